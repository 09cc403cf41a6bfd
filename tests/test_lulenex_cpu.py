"""Lulenex without a GPU: the folder reader and its registry, synthetic parameters, and properties of the plain restatement (lulenex_ref) that the GPU
tests rest on -- also that a planted mistake would show in them."""
import importlib
import itertools
import json

import numpy as np
import pytest

import helpers as H
import lulenex_helpers as LH
import lulenex_ref as L
import suzulix_ref as S
import vilepel_helpers as VH

arch = importlib.import_module("maxtext-indextts2_amd.architectures")


def test_reader_takes_every_size_from_the_folder(tmp_path):
  cfg = LH.mixed_model()
  w = LH.random_weights(cfg)
  c = VH.config(VH.write_model(tmp_path, cfg, w))
  assert (c.vocab_size, c.emb_dim, c.normalization_layer_epsilon, c.decoder_block, c.num_decoder_layers) == (203, 88, 3e-5, "hybrid", 8)
  assert (c.hybrid_norm_kind, c.hybrid_norm_places, c.logits_via_embedding, c.hybrid_streams, c.embedding_scale, c.logit_scale) == (arch.NORM_ONE, arch.NORM_BEFORE, False, 0, 1.0, 1.0)
  l = c.hybrid_layers
  assert [x.number for x in l] == [0, 1, 2, 3, 1, 2, 3, 4] == L.layer_runs(cfg)
  assert [x.weights_of for x in l] == [-1] * 4 + [1, 2, 3, -1]
  assert {i: x.loop_pass for i, x in enumerate(l) if x.loop_pass >= 0} == {1: 0, 4: 1} == L.pass_starts(cfg)
  assert [x.mixer for x in l] == [arch.MIX_SCAN, arch.MIX_ATTENTION, arch.MIX_SCAN, arch.MIX_ATTENTION, arch.MIX_ATTENTION, arch.MIX_SCAN, arch.MIX_ATTENTION, arch.MIX_ATTENTION]
  assert (l[2].inner, l[2].state, l[2].dt_rank, l[2].conv, l[2].ffn, l[2].beside) == (130, 20, 11, 4, arch.FFN_NONE, None)
  assert (l[3].heads, l[3].kv_heads, l[3].dim, l[3].vdim, l[3].rot_dim, l[3].rope_base, l[3].attn_scale, l[3].chunk, l[3].window, l[3].mix_scale) == (4, 1, 30, 30, 30, 5000.0, 0.2, 16, 0, 1.1)
  assert (l[3].rope_pairs, l[3].qk_norm, l[3].sink, l[3].out_gate, l[3].key_values, l[3].mix_bias) == (arch.ROPE_HALVES, arch.QK_NORM_PLAIN, 1, arch.GATE_HEADS, 1, 1)
  b = l[3].beside
  assert (b.mixer, b.heads, b.dim, b.vdim, b.decay, b.mix_scale, b.rot_dim) == (arch.MIX_LIGHTNING, 2, 34, 18, (0.5, 0.9990234375), 0.4, 0)
  assert (l[7].chunk, l[3].ff, l[3].glu) == (0, 33, arch.ACT_XIELU) and all(x.shift for x in l) and all(arch.carries_state(x) for x in l)
  assert arch.parameter_shapes(c) == {k: v.shape for k, v in w.items()}


def test_loops(tmp_path):
  layers = [LH.with_mlp(LH.mamba(), None)] * 3
  for i, (loop, want, starts) in enumerate(((None, [0, 1, 2], {}), ({"start": 0, "stop": 3, "times": 1}, [0, 1, 2], {0: 0}), ({"start": 2, "stop": 3, "times": 3}, [0, 1, 2, 2, 2], {2: 0, 3: 1, 4: 2}),
                                            ({"start": 0, "stop": 2, "times": 2}, [0, 1, 0, 1, 2], {0: 0, 2: 1}))):
    cfg = LH.model(layers, loop=loop)
    c = VH.config(VH.write_model(tmp_path / str(i), cfg, {"embed": np.zeros((2, 2))}))
    assert [x.number for x in c.hybrid_layers] == want == L.layer_runs(cfg)
    assert {j: x.loop_pass for j, x in enumerate(c.hybrid_layers) if x.loop_pass >= 0} == starts == L.pass_starts(cfg)
    assert {k: v for k, v in arch.parameter_shapes(c).items() if k.startswith("loop")} == {k: v for k, v in LH.shapes(cfg).items() if k.startswith("loop")}


def test_synthetic_parameters(tmp_path):
  with open(tmp_path / "config.json", "w", encoding="utf-8") as f:
    json.dump(LH.mixed_model(), f)
  c = VH.config(tmp_path)
  shapes = arch.parameter_shapes(c)
  w = H.synth.synth_weights(c, 3)
  assert {k: v.shape for k, v in w.items()} == shapes
  assert {n: s for n, s, _ in H.synth.device_tree_spec(c)} == shapes


def test_reader_refuses_what_it_does_not_know(tmp_path):
  cfg = LH.mixed_model()
  z = {"embed": np.zeros((2, 2))}
  m = cfg["layers"][1]["mixer"]
  for i, (change, text) in enumerate((({"type": "other"}, "type"), ({"mlp": {"kind": "moe"}}, "kind"), ({"mixer": dict(m, left=dict(m["left"], kv_heads=4))}, "heads"),
                                      ({"mixer": dict(m, left=dict(m["left"], rot={"base": 9.0, "dims": 20}))}, "rotated"), ({"mixer": dict(m, left=dict(m["left"], vdim=20))}, "vdim"),
                                      ({"mixer": dict(m, right=dict(m["right"], decay=[0.5]))}, "decays"))):
    layers = list(cfg["layers"])
    layers[1] = dict(layers[1], **change)
    with pytest.raises(ValueError, match=text):
      VH.config(VH.write_model(tmp_path / str(i), dict(cfg, layers=layers), z))


# ---------------------------------------------------------------------------------------------------- the restatement
def test_scan_against_its_sum_over_the_past():
  rng = np.random.default_rng(1)
  T, C, N = 9, 3, 4
  x, dt, A = rng.standard_normal((T, C)), rng.random((T, C)), -rng.random((C, N))
  B, Y, D = rng.standard_normal((T, N)), rng.standard_normal((T, N)), rng.standard_normal(C)
  y = L.selective_scan(x, dt, A, B, Y, D)
  for t in range(T):
    for c in range(C):
      want = sum((np.exp(A[c] * dt[j + 1:t + 1, c].sum()) * dt[j, c] * x[j, c] * B[j]) @ Y[t] for j in range(t + 1)) + D[c] * x[t, c]
      assert np.isclose(y[t, c], want)


def test_short_convolution_and_shift():
  x = np.arange(5.0)[:, None] + 1
  assert np.allclose(L.short_convolution(x, np.array([[100.0, 10.0, 1.0]]), np.array([0.5]))[:, 0], [1.5, 12.5, 123.5, 234.5, 345.5])
  assert np.allclose(L.token_shift(x, np.array([0.25]))[:, 0], [0.75, 1.75, 2.75, 3.75, 4.75])


def test_xielu_against_its_integral():
  """Its slope is 2 a z + 1/2 above zero and b (exp(z) - 1) + 1/2 below, and it passes through 0."""
  p, q = 0.3, -0.4
  a, b = np.log1p(np.exp(p)), 0.5 + np.log1p(np.exp(q))
  z = np.linspace(-6, 4, 4001)
  slope = np.gradient(L.xielu(z, p, q), z)
  assert np.abs(slope - np.where(z > 0, 2 * a * z, b * (np.exp(z) - 1)) - 0.5)[1:-1].max() < 5e-3 and L.xielu(np.zeros(1), p, q)[0] == 0


def test_chunks_sinks_and_rotated_norms():
  mask = L.seen(7, 3)
  assert mask.sum(1).tolist() == [1, 2, 3, 1, 2, 3, 1] and L.seen(4, None).sum(1).tolist() == [1, 2, 3, 4]
  a = L.sink_softmax(np.zeros((7, 7)), mask, np.log(2.0))
  assert np.allclose(a.sum(1), [1 / 3, 2 / 4, 3 / 5, 1 / 3, 2 / 4, 3 / 5, 1 / 3])
  x = np.random.default_rng(0).standard_normal((5, 12))
  rot = {"base": 50.0, "dims": 8}
  assert np.allclose(L.rms(L.rotate_halves(x, np.arange(5.0), rot), 0.1), L.rotate_halves(L.rms(x, 0.1), np.arange(5.0), rot))


def test_restatement_is_causal():
  cfg = LH.mixed_model()
  w = LH.random_weights(cfg, 1)
  t = VH.tokens(cfg, 40, 2)
  assert np.allclose(L.forward(cfg, w, t[:23]), L.forward(cfg, w, t)[:23], atol=1e-10)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_planted_mistakes_would_show(dtype, monkeypatch):
  """Each mistake moves the logits of the model that the GPU tests run by more than their tolerance."""
  cfg = LH.mixed_model()
  w = LH.random_weights(cfg, 5)
  t = VH.tokens(cfg, 80, 6)
  good = L.forward(cfg, w, t)
  att, lig, mam, scan, enter, ret = L.chunked_attention, L.lightning, L.mamba, L.selective_scan, L.enter_pass, L.retention_states
  zero = lambda *parts: {k: np.zeros_like(v) if any(k.endswith(p) for p in parts) else v for k, v in w.items()}
  ones = lambda part: {k: np.ones_like(v) if k.endswith(part) else v for k, v in w.items()}

  def par(l=att, r=lig, f=lambda m: m):
    return {"MIXERS": dict(L.MIXERS, parallel=lambda h, u, m, e: f(m)["left_scale"] * l(h, L.under(u, "left."), m["left"], e) + f(m)["right_scale"] * r(h, L.under(u, "right."), m["right"], e))}

  def normed_values(h, u, m, e):
    """The values after norm and rotation instead of before."""
    T, G, d, pos = len(h), m["kv_heads"], m["dim"], np.arange(len(h), dtype=np.float64)
    k = (L.linear(u["k"], h) + u["k.b"]).reshape(T, G, d)
    v = np.stack([L.rms(L.rotate_halves(k[:, g], pos, m["rot"]), e) for g in range(G)], 1)
    soft = L.sink_softmax
    rows, out = [], np.empty((T, m["heads"], d))
    with monkeypatch.context() as inner:
      inner.setattr(L, "sink_softmax", lambda s, mask, sink: rows.append(soft(s, mask, sink)) or rows[-1])
      att(h, u, m, e)
    for i in range(m["heads"]):
      out[:, i] = L.sigmoid(L.linear(u["g"], h))[:, i:i + 1] * (rows[i] @ v[:, i // (m["heads"] // G)])
    return L.linear(u["o"], out.reshape(T, -1)) + u["o.b"]

  def no_norms(h, u, m, e):
    with monkeypatch.context() as inner:
      inner.setattr(L, "rms", lambda x, e: x)
      return att(h, u, m, e)

  mistakes = {
      "chunk a token longer": dict(seen=lambda T, n, f=L.seen: f(T, n and n + 1)), "no chunks": dict(seen=lambda T, n, f=L.seen: f(T, None)),
      "a window for a chunk": dict(seen=lambda T, n, f=L.seen: f(T, None) & ((np.arange(T)[:, None] - np.arange(T)[None]) < (n or T))),
      "neighbours for halves": dict(rotate_halves=S.rotate_neighbours),
      "nothing turns": dict(rotate_halves=lambda x, p, r: x), "no sinks": dict(sink_softmax=lambda s, m, k, f=L.sink_softmax: f(s, m, -1e9)),
      "sinks scaled": par(l=lambda h, u, m, e: att(h, dict(u, sink=u["sink"] * m["scale"]), m, e)),
      "no query and key norms": par(l=no_norms), "no key bias": zero("left.k.b"), "no query bias": zero("left.q.b"), "no output bias": zero("left.o.b"), "no head gates": zero("left.g"), "values after the norm": par(l=normed_values),
      "heads on the wrong key head": par(l=lambda h, u, m, e: att(h, dict(u, k=np.roll(u["k"], m["dim"], 0), **{"k.b": np.roll(u["k.b"], m["dim"], 0)}), m, e) if m["kv_heads"] > 1 else att(h, u, m, e)),
      "output bias not scaled": {k: v / 0.8 if k == "l1.mix.left.o.b" else v for k, v in w.items()},
      "left alone": par(r=lambda h, u, m, e: 0.0), "right alone": par(l=lambda h, u, m, e: 0.0), "scales swapped": par(f=lambda m: {"left_scale": m["right_scale"], "right_scale": m["left_scale"]}),
      "decays swapped": par(r=lambda h, u, m, e: lig(h, u, dict(m, decay=m["decay"][::-1]), e)), "state lost": dict(retention_states=lambda q, k, v, d: (q * k).sum(1, keepdims=True) * v),
      "read before written": dict(retention_states=lambda q, k, v, d: ret(q, k, v, d) - (q * k).sum(1, keepdims=True) * v),
      "norm per head": par(r=lambda h, u, m, e: lig(h, u, m, e) * 0 + L.linear(u["o"], np.concatenate([L.rms(x, e) for x in np.split(
          np.concatenate([ret(*(L.silu(L.linear(u[n], h)).reshape(len(h), m["heads"], -1)[:, i] for n in ("q", "k", "v")), m["decay"][i]) for i in range(m["heads"])], 1), m["heads"], 1)], 1)
          * u["norm"] * L.sigmoid(L.linear(u["g"], h)))),
      "no lightning norm weight": ones("right.norm"), "no lightning gate": zero("right.g"),
      "scan state lost": dict(selective_scan=lambda x, d, A, B, C, D: d * x * (B * C).sum(1, keepdims=True) + D * x), "scan without decay": dict(selective_scan=lambda x, d, A, B, C, D: scan(x, d, 0 * A, B, C, D)),
      "no skip": zero("mix.D"), "one rate for all states": dict(selective_scan=lambda x, d, A, B, C, D: scan(x, d, A[:, :1] + 0 * A, B, C, D)), "B and C swapped": dict(selective_scan=lambda x, d, A, B, C, D: scan(x, d, A, C, B, D)),
      "no step size bias": zero("mix.dt.b"), "no convolution bias": zero("conv.b"), "taps reversed": {k: v[:, ::-1] if k.endswith(".conv") else v for k, v in w.items()},
      "x and z swapped": {k: np.roll(v, len(v) // 2, 0) if k.endswith("mix.in") else v for k, v in w.items()},
      "no shift": zero(".shift"), "shift of the shifted": dict(token_shift=lambda h, mu: np.stack(list(itertools.accumulate(h, lambda a, b: b + (a - b) * mu)))),
      "first token shifts from itself": dict(token_shift=lambda h, mu: h + (np.concatenate([h[:1], h[:-1]]) - h) * mu),
      "no steps": zero("loop.step"), "first step twice": {k: np.repeat(v[:1], len(v), 0) if k == "loop.step" else v for k, v in w.items()},
      "input halves swapped": dict(enter_pass=lambda x, x0, W, s: enter(x0, x, W, s)), "stream kept": dict(enter_pass=lambda x, x0, W, s: x + s), "no embedding output": dict(enter_pass=lambda x, x0, W, s: enter(x, 0 * x0, W, s)),
      "step before the product": dict(enter_pass=lambda x, x0, W, s: enter(x + s, x0, W, 0 * s)),
      "unit numbers swapped": {k: v[::-1] if k.endswith("mlp.act") else v for k, v in w.items()}, "relu squared": dict(xielu=lambda z, p, q: np.maximum(z, 0) ** 2),
      "no loop": dict(layer_runs=lambda c: list(range(len(c["layers"])))), "norms of one": ones("norm1"),
  }
  for name, change in mistakes.items():
    with monkeypatch.context() as mp:
      if "embed" in change:
        bad = L.forward(cfg, change, t)
      else:
        for k, f in change.items():
          mp.setattr(L, k, f)
        bad = L.forward(cfg, w, t)
    r = LH.rel(bad, good)
    worst = r[0] if "first token" in name else np.quantile(r[5:], 0.9)
    print(dtype, name, worst)
    assert worst > LH.TOL[dtype] * (1.5 if dtype == "float32" else 1.0), (name, worst)
