"""Lulenex on the GPU against the plain float64 restatement (lulenex_ref): every mechanism alone at many sizes, then the cache, the states, the batch and
the engine's entry points.  float32 is held to rounding of f32 sums, bfloat16 to rounding of its operands (lulenex_helpers.TOL)."""
import contextlib
import ctypes
import dataclasses
import importlib
import io
import json
import sys

import numpy as np
import pytest
import torch

import helpers as H
import lulenex_helpers as LH
import lulenex_ref as L
import vilepel_helpers as VH

pytestmark = pytest.mark.gpu
DTYPES = ["float32", "bfloat16"]


def residuals(eng, cfg, toks, cuts, runs):
  """The residual stream behind every layer run [tokens, runs width], the tokens fed in portions."""
  s, got, at, i = VH.scheduler(eng), [], 0, 0
  while at < len(toks):
    m = min(cuts[min(i, len(cuts) - 1)], len(toks) - at)
    tap = torch.zeros(runs * m * cfg["width"], device="cuda")
    H.lib.check(eng.lib.ixt_set_residual_tap(eng._ctx, ctypes.c_void_p(tap.data_ptr()), tap.numel()))
    s.step([("r", toks[at:at + m], [])])
    got.append(tap.cpu().numpy().reshape(runs, m, -1).transpose(1, 0, 2).reshape(m, -1))
    at, i = at + m, i + 1
  s.release("r")
  H.lib.check(eng.lib.ixt_set_residual_tap(eng._ctx, None, 0))
  return np.concatenate(got)


def one_layer(tmp_path, layer, dtype, n=50, seed=0, portions=(), alter=None, loop=None, **kw):
  """The residual stream behind one layer (every pass of it) for a prompt and for the same tokens in portions against the restatement."""
  cfg = LH.model([layer], loop=loop)
  w = LH.random_weights(cfg, seed)
  w["embed"] = w["embed"] / 3                       # the layer's part of the stream counts as much as what it joins
  if alter is not None:
    alter(w)
  w = LH.rounded(w)
  toks = VH.tokens(cfg, n, seed + 1)
  taps = []
  L.forward(cfg, w, toks, taps)
  want = np.concatenate(taps, axis=1)
  eng, _ = VH.engine(VH.write_model(tmp_path, cfg, w), dtype=dtype, **kw)
  for cuts in ((n,),) + tuple(portions):
    r = LH.rel(residuals(eng, cfg, toks, cuts, len(taps)), want)
    if dtype == "float32":
      assert r.max() < 1e-5, (cuts, int(r.argmax()), r.max())
    else:
      assert np.quantile(r, 0.9) < 0.015 and r.max() < 0.03, (cuts, int(r.argmax()), np.quantile(r, 0.9), r.max())
  eng.close()


P, lf, rt = LH.parallel, LH.left, LH.right
MIXERS = {
    "parallel: one head each": P(lf(heads=1, kv_heads=1, dim=8, dims=8), rt(heads=1, dim=8, vdim=8)),
    "parallel: odd sizes": P(lf(heads=3, kv_heads=3, dim=23, dims=10), rt(heads=5, dim=23, vdim=17)),
    "parallel: nothing turns": P(lf(heads=2, kv_heads=2, dims=0)),
    "parallel: one pair turns": P(lf(heads=4, kv_heads=2, dims=2), rt(heads=2)),
    "parallel: everything turns": P(lf(heads=4, kv_heads=1, dim=30, dims=30), rt(heads=4, dim=30, vdim=16)),
    "parallel: many heads on one": P(lf(heads=20, kv_heads=1, dim=12, dims=12), rt(heads=7, dim=9, vdim=5)),
    "parallel: more heads than a tile": P(lf(heads=70, kv_heads=2, dim=8, dims=4)),
    "parallel: 32 and values wider": P(lf(heads=6, kv_heads=2, dim=32, dims=16), rt(heads=2, dim=40, vdim=128)),
    "parallel: 64 and keys wider": P(lf(heads=4, kv_heads=4, dim=64, dims=64, scale=0.1), rt(heads=2, dim=130, vdim=20)),
    "parallel: 90": P(lf(heads=4, kv_heads=1, dim=90, dims=64, scale=0.1), rt(heads=3, dim=64, vdim=62)),
    "parallel: 128 and 200": P(lf(heads=4, kv_heads=2, dim=128, dims=64, scale=0.09), rt(heads=2, dim=128, vdim=200)),
    "parallel: 180 and 300": P(lf(heads=2, kv_heads=1, dim=180, dims=64, scale=0.08), rt(heads=1, dim=260, vdim=300)),
    "parallel: beyond the tiles": P(lf(heads=2, kv_heads=1, dim=300, dims=64, scale=0.05), rt(heads=3, dim=20, vdim=500)),
    "parallel: no chunks": P(lf(chunk=None)),
    "parallel: chunks of one": P(lf(chunk=1)),
    "parallel: chunks of two": P(lf(chunk=2)),
    "parallel: chunks of a tile": P(lf(chunk=64)),
    "parallel: one chunk": P(lf(chunk=1000)),
    "parallel: sharp scores": P(lf(scale=2.5)),
    "parallel: fast and not at all": P(r=rt(heads=3, decay=[0.05, 0.75, 1.0])),
    "parallel: factors of one": P(left_scale=1.0, right_scale=1.0),
    "parallel: factors far apart": P(left_scale=0.03, right_scale=2.5),
    "scan: one of each": LH.mamba(inner=1, state=1, dt_rank=1, conv=1),
    "scan: odd sizes": LH.mamba(inner=67, state=5, dt_rank=3, conv=2),
    "scan: 16 states": LH.mamba(inner=128, state=16, dt_rank=8, conv=4),
    "scan: 32 states": LH.mamba(inner=200, state=32, dt_rank=130, conv=4),
    "scan: 33 states": LH.mamba(inner=72, state=33, dt_rank=16, conv=5),
    "scan: 100 states": LH.mamba(inner=40, state=100, dt_rank=5, conv=4),
    "scan: 200 states": LH.mamba(inner=36, state=200, dt_rank=9, conv=7),
    "scan: many channels": LH.mamba(inner=1100, state=12, dt_rank=40, conv=4),
}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(MIXERS))
def test_mixer_alone(tmp_path, name, dtype):
  one_layer(tmp_path, LH.with_mlp(MIXERS[name], None), dtype, n=75, portions=((1,), (2,), (33, 2), (7, 1, 40), (64, 11)))


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_looped_layer_keeps_a_state_per_pass(tmp_path, dtype):
  for i, layer in enumerate((LH.parallel(), LH.mamba())):
    for times in (1, 3):
      one_layer(tmp_path / f"{i}{times}", LH.with_mlp(layer, None), dtype, n=40, portions=((1,), (9, 31)), loop={"start": 0, "stop": 1, "times": times})


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("ff", [1, 60, 128, 300])
def test_units(tmp_path, ff, dtype):
  """Products far on both sides of zero and close to it."""
  for i, f in enumerate((0.02, 1.0, 2.5)):
    def spread(w, f=f):
      w["l0.mlp.up"] *= f
      w["l0.mlp.down"] *= 0.5 / max(f, 1.0) ** 2
    one_layer(tmp_path / str(i), LH.with_mlp(LH.mamba(), LH.dense(ff)), dtype, n=70, portions=((1,), (9, 61)), alter=spread)


@pytest.mark.parametrize("dtype", DTYPES)
def test_token_shift(tmp_path, dtype):
  """No shift, the previous token only, and beyond; portions of one and two tokens, so that what is kept is all there is."""
  for i, mu in enumerate((0.0, 1.0, 2.0)):
    def all_alike(w, mu=mu):
      w["l0.shift"][:] = mu
    one_layer(tmp_path / str(i), LH.with_mlp(LH.parallel(), LH.dense()), dtype, n=30, portions=((1,), (2,), (3, 1)), alter=all_alike)


@pytest.mark.parametrize("dtype", DTYPES)
def test_sinks_and_step_sizes_from_weak_to_strong(tmp_path, dtype):
  for i, sink in enumerate((-30.0, 6.0)):
    def sinks(w, sink=sink):
      w["l0.mix.left.sink"][:] = sink
    one_layer(tmp_path / f"s{i}", LH.with_mlp(LH.parallel(), None), dtype, n=40, portions=((1,), (21, 2)), alter=sinks)
  for i, b in enumerate((-9.0, 2.5)):               # step sizes of 1e-4, and of some units: decays down to nothing
    def steps(w, b=b):
      w["l0.mix.dt.b"][:] = b
    one_layer(tmp_path / f"d{i}", LH.with_mlp(LH.mamba(), None), dtype, n=90, seed=4, portions=((1,), (65, 2)), alter=steps)


@pytest.mark.parametrize("dtype", DTYPES)
def test_many_rows_take_the_prompt_kernels(tmp_path, dtype):
  """300 rows in one pass: the ring GEMMs, tall attention tiles, several chunks of the recurrences."""
  for i, layer in enumerate((LH.with_mlp(LH.parallel(lf(chunk=70)), LH.dense()), LH.with_mlp(LH.parallel(lf(heads=8, kv_heads=2, dim=60, dims=60, scale=0.1, chunk=None), rt(heads=2, dim=90, vdim=100,
                             decay=[0.97, 1 - 2.0 ** -10])), None), LH.with_mlp(LH.mamba(inner=150, state=16, conv=4), LH.dense(260)), LH.with_mlp(LH.mamba(inner=80, state=40, dt_rank=20), None))):
    one_layer(tmp_path / str(i), layer, dtype, n=300, portions=((150, 129, 1),), target=320, rows=320, pages=40)


@pytest.mark.parametrize("dtype", DTYPES)
def test_no_decoder_sizes_are_special(tmp_path, dtype):
  for i, kw in enumerate((dict(vocab=17, width=33, eps=1e-3), dict(vocab=1500, width=130, eps=1e-6), dict(vocab=300, width=2050), dict(vocab=300, width=2052), dict(vocab=100, width=4100))):
    cfg = LH.model([LH.with_mlp(LH.parallel(), None), LH.with_mlp(LH.mamba(), LH.dense())], loop={"start": 1, "stop": 2, "times": 2} if i % 2 else {"start": 0, "stop": 2, "times": 1}, **kw)
    w = LH.random_weights(cfg, i)
    eng, _ = VH.engine(VH.write_model(tmp_path / str(i), cfg, w), dtype=dtype)
    t = VH.tokens(cfg, 20, i)
    LH.check(VH.run_portions(VH.scheduler(eng), "r", t, (17, 1)), L.forward(cfg, w, t), dtype, kw)
    eng.close()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("loop", [None, {"start": 0, "stop": 3, "times": 1}, {"start": 0, "stop": 3, "times": 2}, {"start": 2, "stop": 3, "times": 3}, {"start": 1, "stop": 2, "times": 2}])
def test_loops(tmp_path, loop, dtype):
  cfg = LH.model([LH.with_mlp(LH.mamba(), LH.dense()), LH.with_mlp(LH.parallel(), None), LH.with_mlp(LH.parallel(lf(chunk=9)), LH.dense())], loop=loop)
  w = LH.random_weights(cfg, 4)
  eng, _ = VH.engine(VH.write_model(tmp_path, cfg, w), dtype=dtype)
  t, taps = VH.tokens(cfg, 60, 1), []
  want, s = L.forward(cfg, w, t, taps), VH.scheduler(eng)
  for cuts in ((60,), (1,), (31, 2)):
    LH.check(VH.run_portions(s, "r", t, cuts), want, dtype, cuts)
    s.release("r")
  r = LH.rel(residuals(eng, cfg, t, (40, 20), len(taps)), np.concatenate(taps, axis=1))      # every run's residual, also the one in front of a pass
  assert r.max() < (1e-5 if dtype == "float32" else 0.02), r.max()
  eng.close()


def test_the_same_switches_in_other_designs(tmp_path, monkeypatch):
  """Two attentions side by side, retention beside lightning attention, chunks and one-number norms without shift and bias, a shift in front of the gated
  delta rule: against the equations written out here."""
  import suzulix_ref as S
  arch = importlib.import_module("maxtext-indextts2_amd.architectures")
  E, V, eps, H_ = 88, 203, 3e-5, arch.HybridLayer
  rng = np.random.default_rng(0)
  rot = {"base": 300.0, "dims": 8}
  one = dict(mixer=arch.MIX_ATTENTION, heads=4, kv_heads=2, dim=20, vdim=20, rot_dim=8, rope_base=300.0, rope_pairs=arch.ROPE_HALVES, attn_scale=0.3, key_values=1)
  runs = (H_(**dict(one, chunk=9, out_gate=arch.GATE_HEADS, mix_scale=0.7), beside=H_(**dict(one, heads=2, vdim=12, key_values=0, out_gate=arch.GATE_FEATURES, mix_scale=1.4))),
          H_(mixer=arch.MIX_RETENTION, heads=2, dim=16, vdim=10, rot_dim=8, rope_base=300.0, rope_pairs=arch.ROPE_HALVES, decay=(0.9, 0.98), mix_scale=1.5, shift=1,
             beside=H_(mixer=arch.MIX_LIGHTNING, heads=3, dim=8, vdim=6, decay=(0.5, 0.9, 0.99))))
  keys = {"decoder_block": "hybrid", "vocab_size": V, "base_emb_dim": E, "base_num_decoder_layers": 2, "normalization_layer_epsilon": eps, "hybrid_norm_kind": arch.NORM_ONE,
          "hybrid_norm_places": arch.NORM_BEFORE, "hybrid_layers": runs}
  monkeypatch.setitem(arch.ARCHITECTURES, "LulenexVariant", lambda c, shapes: keys)
  names = arch.parameter_shapes(VH.config(VH.write_model(tmp_path / "0", {"architecture": "LulenexVariant"}, {"embed": np.zeros((2, 2))})))
  w = LH.rounded({n: rng.standard_normal(s) / (np.sqrt(s[-1]) if len(s) == 2 and n != "embed" else 1.0) + (1.0 if "norm" in n else 0.0) for n, s in names.items()})

  def attention(h, u, m):
    T, pos, out = len(h), np.arange(len(h), dtype=np.float64), []
    k = S.linear(u["k"], h).reshape(T, 2, 20)
    v = k if m.key_values else S.linear(u["v"], h).reshape(T, 2, 12)
    q = S.linear(u["q"], h).reshape(T, m.heads, 20)
    gate = S.sigmoid(S.linear(u["g"], h)).reshape(T, m.heads, -1)
    for i in range(m.heads):
      g = i // (m.heads // 2)
      s = S.rotate_halves(q[:, i], pos, rot) @ S.rotate_halves(k[:, g], pos, rot).T * 0.3
      out.append(S.causal_softmax(np.where(L.seen(T, m.chunk or None), s, -np.inf)) @ v[:, g] * gate[:, i])
    return S.linear(u["o"], np.concatenate(out, axis=1))

  t = VH.tokens({"vocab": V}, 50, 3)
  x = w["embed"][t]
  h = L.one_number_norm(x, w["l0.norm1"], eps)
  x = x + 0.7 * attention(h, S.under(w, "l0.mix.left."), runs[0]) + 1.4 * attention(h, S.under(w, "l0.mix.right."), runs[0].beside)
  h = L.token_shift(L.one_number_norm(x, w["l1.norm1"], eps), w["l1.shift"])
  x = x + 1.5 * S.retention(h, S.under(w, "l1.mix.left."), {"heads": 2, "dim": 16, "vdim": 10, "rot": rot, "decay": runs[1].decay}, eps)
  x = x + L.lightning(h, S.under(w, "l1.mix.right."), {"heads": 3, "dim": 8, "vdim": 6, "decay": runs[1].beside.decay}, eps)
  want = S.linear(w["head"], L.one_number_norm(x, w["final.norm"], eps))
  for dtype in DTYPES:
    eng, _ = VH.engine(VH.write_model(tmp_path / dtype, {"architecture": "LulenexVariant"}, w), dtype=dtype)
    s = VH.scheduler(eng)
    for cuts in ((50,), (1,), (17, 2)):
      LH.check(VH.run_portions(s, "r", t, cuts), want, dtype, cuts)
      s.release("r")
    eng.close()
  refused = dataclasses.replace(runs[0], beside=H_(mixer=arch.MIX_SCAN, inner=4, state=4))
  monkeypatch.setitem(arch.ARCHITECTURES, "LulenexVariant", lambda c, shapes: dict(keys, hybrid_layers=(refused,), base_num_decoder_layers=1))
  with pytest.raises(NotImplementedError, match="side by side"):
    VH.engine(VH.write_model(tmp_path / "1", {"architecture": "LulenexVariant"}, {"embed": np.zeros((2, 2))}))


# ---------------------------------------------------------------------------------------------------- far tokens that random weights would hide
def marked_model(kind, rng, chunk=None, eps=3e-5):
  """One layer in which one marked token stands out for every later position, whatever the distance -> (cfg, weights, the mark)."""
  layer = {"attention": P(lf(heads=4, kv_heads=2, dim=32, dims=4, scale=1.0, chunk=chunk)), "lightning": P(lf(heads=1, kv_heads=1, dim=4, dims=4), rt(heads=4, dim=16, vdim=16, decay=[1 - 2.0 ** -12,
           1 - 2.0 ** -11, 1 - 2.0 ** -10, 1.0])), "scan": LH.mamba(inner=40, state=12, dt_rank=4, conv=3)}[kind]
  cfg = LH.model([LH.with_mlp(layer, None)], eps=eps)
  w, mark, E = LH.random_weights(cfg, 3), 7, cfg["width"]
  common, special = np.arange(E) < 12, (np.arange(E) >= 12) & (np.arange(E) < 24)
  sign = np.sign(rng.standard_normal(E))
  w["embed"] /= 3
  w["embed"][:, common] = 2.0 * sign[common]               # every token has this, only the mark has that
  w["embed"][:, special] = 0.0
  w["embed"][mark, special] = 3.0 * sign[special]
  w["l0.shift"] *= 0.1

  def point(name, rows, direction, feats, gain, noise=0.15):
    """The named matrix: small on the two groups of features, `direction` (of `rows`) for what is in `feats`."""
    m = noise * w[name].reshape(-1, rows, E)
    m[:, :, common | special] = 0.0
    m[:, :, feats] += gain * direction[None, :, None] * sign[None, None, feats] / 12
    w[name] = m.reshape(w[name].shape)

  if kind == "attention":
    q = rng.standard_normal(32)
    q[:4] = 0.0
    q /= np.linalg.norm(q)
    point("l0.mix.left.q", 32, q, common, 5.0)
    point("l0.mix.left.k", 32, q, special, 12.0, 0.4)
    w["l0.mix.right.o"] *= 0.0
  elif kind == "lightning":
    q = np.abs(rng.standard_normal(16))
    q /= np.linalg.norm(q)
    point("l0.mix.right.q", 16, q, common, 5.0)
    point("l0.mix.right.k", 16, q, special, 60.0)
    w["l0.mix.left.o"] *= 0.0
  else:                                                    # channels 0 .. 7 speak of every token, 8 .. 15 of the mark: B takes these, C those
    m = 0.15 * w["l0.mix.in"]
    m[:40][:, common | special] = 0.0
    m[:8, common] += 3.0 * sign[common] / 12
    m[8:16, special] += 8.0 * sign[special] / 12
    w["l0.mix.in"] = m
    w["l0.mix.conv"] = np.array([0.05, 0.1, 1.0]) + 0.0 * w["l0.mix.conv"]
    w["l0.mix.conv.b"] *= 0.0
    b = 0.05 * w["l0.mix.x"]
    b[4:16, 8:16] += 0.3
    b[16:28, :8] += 0.2
    w["l0.mix.x"] = b
    w["l0.mix.A_log"] = np.log(1e-3) + 0.2 * w["l0.mix.A_log"]
    w["l0.mix.dt"] *= 0.1
  return cfg, LH.rounded(w), mark


def shows(cfg, w, t, place, rows):
  """The mark at `place` can be told from another token in `rows` by more than the tolerance."""
  u = t.copy()
  u[place] = 8
  r = LH.rel(L.forward(cfg, w, u), L.forward(cfg, w, t))[rows]
  assert r.min() > 3 * LH.TOL["bfloat16"], r.min()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind", ["attention", "lightning", "scan"])
def test_far_tokens_stand_out(tmp_path, dtype, kind):
  """A marked token hundreds of positions back, at the start, next to page, tile and chunk borders, seen from the end of a long prompt and from decoded
  tokens (keys in several splits)."""
  n = 500
  cfg, w, mark = marked_model(kind, np.random.default_rng(6))
  eng, params = VH.engine(VH.write_model(tmp_path, cfg, w), dtype=dtype, slots=1, pages=80, target=520, rows=520)
  for place in (0, 1, 63, 64, 255, 300):
    t = VH.tokens(cfg, n, 9)
    t[t == mark] = 8
    t[place] = mark
    want = L.forward(cfg, w, t)
    shows(cfg, w, t, place, slice(-20, None))
    for cuts in ((n,), (n - 9, 1), (257, 129, 31, 2)):
      s = VH.scheduler(eng)
      LH.check(VH.run_portions(s, "r", t, cuts), want, dtype, (place, cuts))
      s.release("r")
    st = eng.init_decode_state(materialize_logits=True)    # the decode step's own kernels
    padded = np.zeros(eng.max_prefill_length, np.int32)
    padded[:n] = t
    prefix, first = eng.prefill(params=params, padded_tokens=padded, true_length=n, slot=0)
    st = eng.insert(prefix, st, 0)
    st, _ = eng.generate(params, st)
    seq = np.concatenate([t, [int(first.data[0, 0])]])
    LH.check(np.concatenate([prefix["logits"].cpu().numpy().reshape(1, -1), st["logits"].cpu().numpy().reshape(1, -1)]), L.forward(cfg, w, seq)[-2:], dtype, (place, "step"))
    eng.release_pages(0)
  eng.close()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("chunk", [37, 64, 100])
def test_chunk_edges(tmp_path, dtype, chunk):
  """A marked token just inside and just outside the chunk of the positions behind it, in prompts, in portions that are cut at and around the edge, and in
  decoding across it."""
  cfg, w, mark = marked_model("attention", np.random.default_rng(6), chunk=chunk)
  n, edge = 3 * chunk - 2, 2 * chunk
  eng, params = VH.engine(VH.write_model(tmp_path, cfg, w), dtype=dtype, slots=2, pages=90, target=320, rows=320)
  for place in (edge - 1, edge, edge + 1, edge - chunk):
    t = VH.tokens(cfg, n, 9)
    t[t == mark] = 8
    t[place] = mark
    want = L.forward(cfg, w, t)
    if place >= edge:
      shows(cfg, w, t, place, slice(-20, None))
    else:                                                  # unseen behind the edge (but for the token shift): a longer chunk would show
      with pytest.MonkeyPatch.context() as mp:
        mp.setattr(L, "seen", lambda T, size, f=L.seen: f(T, size) | (L.np.tril(np.ones((T, T), bool)) & (np.arange(T)[None] == place)))
        assert LH.rel(L.forward(cfg, w, t), want)[edge + 2:edge + 20].min() > 3 * LH.TOL["bfloat16"]
    for cuts in ((n,), (edge, 1), (edge - 1, 2), (edge + 1, 5), (edge - 3, 1)):
      s = VH.scheduler(eng)
      LH.check(VH.run_portions(s, "r", t, cuts), want, dtype, (place, cuts))
      s.release("r")
    k = edge - 2                                           # the decode step across the edge
    st = eng.init_decode_state(materialize_logits=True)
    padded = np.zeros(eng.max_prefill_length, np.int32)
    padded[:k] = t[:k]
    prefix, first = eng.prefill(params=params, padded_tokens=padded, true_length=k, slot=0)
    st, seq, got = eng.insert(prefix, st, 0), list(t[:k]) + [int(first.data[0, 0])], []
    for _ in range(6):
      st, r = eng.generate(params, st)
      got.append(st["logits"].cpu().numpy()[0].reshape(-1).copy())
      seq.append(int(r.data[0, 0]))
    LH.check(np.stack(got), L.forward(cfg, w, seq[:-1])[-6:], dtype, (place, "step"))
    eng.release_pages(0)
  eng.close()


# ---------------------------------------------------------------------------------------------------- cache and batches
@pytest.fixture(scope="module", params=DTYPES)
def whole(request, tmp_path_factory):
  cfg = LH.mixed_model()
  w = LH.random_weights(cfg, 5)
  eng, params = VH.engine(VH.write_model(tmp_path_factory.mktemp("lulenex"), cfg, w), dtype=request.param, slots=3, pages=30)
  yield cfg, w, eng, params, request.param
  eng.close()


def test_prompt_token_by_token_and_portions(whole):
  cfg, w, eng, _, dtype = whole
  t = VH.tokens(cfg, 80, 6)
  want = L.forward(cfg, w, t)
  s, base = VH.scheduler(eng), None
  for cuts in ((80,), (1,), (2,), (3, 5), (16,), (17, 1, 2, 30), (79, 1)):
    got = VH.run_portions(s, "r", t, cuts)
    LH.check(got, want, dtype, cuts)
    if base is None:
      base = got
    elif dtype == "float32":                     # and among themselves, beyond the restatement
      assert VH.rel(got, base).max() < 3e-5, cuts
    s.release("r")


def test_first_tokens(whole):
  cfg, w, eng, _, dtype = whole
  s = VH.scheduler(eng)
  for n in (1, 2, 3, 4):
    t = VH.tokens(cfg, n, 20 + n)
    LH.check(VH.run_portions(s, "r", t, (n,)), L.forward(cfg, w, t), dtype, n)
    s.release("r")


def test_unequal_requests_in_one_batch(whole):
  """Prompts, portions and single tokens of three requests in every step, one request paused for some steps."""
  cfg, w, eng, _, dtype = whole
  toks = {"a": VH.tokens(cfg, 70, 48), "b": VH.tokens(cfg, 33, 62), "c": VH.tokens(cfg, 52, 48)}
  sizes = [20, 1, 1, 31, 2, 2, 17, 1]
  s, at, got, step = VH.scheduler(eng), dict.fromkeys(toks, 0), {k: [] for k in toks}, 0
  while any(at[k] < len(toks[k]) for k in toks):
    entries = []
    for i, k in enumerate(toks):
      if (step + i) % 4 == 3 or at[k] == len(toks[k]):
        continue
      n = min(sizes[(step * 3 + i) % len(sizes)], len(toks[k]) - at[k])
      entries.append((k, toks[k][at[k]:at[k] + n], list(range(n))))
      at[k] += n
    step += 1
    if not entries:
      continue
    lg = s.step(entries)[0].cpu().numpy()
    for k, x, _ in entries:
      got[k].append(lg[:len(x)])
      lg = lg[len(x):]
  for k in toks:
    LH.check(np.concatenate(got[k]), L.forward(cfg, w, toks[k]), dtype, k)
    s.release(k)


@pytest.mark.parametrize("dtype", DTYPES)
def test_slots_and_pages_are_used_again(tmp_path, dtype):
  """A pool for one and a half requests and two slots: every new request takes pages that another one has left full."""
  cfg = LH.mixed_model()
  w = LH.random_weights(cfg, 8)
  eng, _ = VH.engine(VH.write_model(tmp_path, cfg, w), dtype=dtype, slots=2, pages=9, page=8, target=64, rows=64)
  s = VH.scheduler(eng)
  for i, (n, cuts) in enumerate(((48, (48,)), (5, (1,)), (33, (9,)), (64, (30, 1)), (2, (2,)), (40, (39, 1)))):
    t = VH.tokens(cfg, n, 40 + i)
    LH.check(VH.run_portions(s, i, t, cuts), L.forward(cfg, w, t), dtype, i)
    s.release(i)
  t = VH.tokens(cfg, 60, 50)
  with pytest.raises(ValueError, match="pool"):
    s.step([("x", t, []), ("y", t, [])])
  eng.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_large_mixed_steps_and_passes(tmp_path, dtype):
  """Steps of some hundred rows made of long portions beside single tokens, also where a step is cut into passes of 128 rows."""
  cfg = LH.mixed_model()
  w = LH.random_weights(cfg, 5)
  path = VH.write_model(tmp_path, cfg, w)
  for rows in (512, 128):
    eng, _ = VH.engine(path, dtype=dtype, slots=4, pages=110, target=256, rows=rows)
    toks = {k: VH.tokens(cfg, n, 100 + n) for k, n in (("a", 250), ("b", 131), ("c", 9), ("d", 200))}
    s, at, got = VH.scheduler(eng), dict.fromkeys(toks, 0), {k: [] for k in toks}
    for sizes in ((("a", 1), ("c", 5), ("b", 130)), (("a", 150), ("b", 1), ("d", 129), ("c", 1)), (("d", 70), ("c", 3), ("a", 98)), (("a", 1), ("d", 1))):
      lg = s.step([(k, toks[k][at[k]:at[k] + n], list(range(n))) for k, n in sizes])[0].cpu().numpy()
      for k, n in sizes:
        got[k].append(lg[:n])
        lg, at[k] = lg[n:], at[k] + n
    for k in toks:
      assert at[k] == len(toks[k])
      LH.check(np.concatenate(got[k]), L.forward(cfg, w, toks[k]), dtype, (rows, k))
    eng.close()


# ---------------------------------------------------------------------------------------------------- the framework's own entry points
def decode_greedy(eng, params, prompt, n, slot=0):
  padded = np.zeros(eng.max_prefill_length, np.int32)
  padded[:len(prompt)] = prompt
  prefix, first = eng.prefill(params=params, padded_tokens=padded, true_length=len(prompt), slot=slot)
  state = eng.insert(prefix, eng.init_decode_state(), slot)
  out = [int(first.data[0, 0])]
  while len(out) < n:
    state, r = eng.generate(params, state)
    out.append(int(r.data[slot, 0]))
  eng.release_pages(slot)
  return np.array(out, np.int32)


def assert_greedy(out, logits, margin=1e-3):
  """The tokens are the argmax of the restatement's logits wherever its lead is not within rounding."""
  top = np.sort(logits, axis=1)
  clear = top[:, -1] - top[:, -2] > margin
  assert clear.mean() > 0.9 and (np.asarray(out)[clear] == logits.argmax(axis=1)[clear]).all()


def test_long_decoding(tmp_path):
  """400 decoded tokens through the engine's decode step: far beyond every window, pages taken one by one."""
  cfg = LH.mixed_model()
  w = LH.random_weights(cfg, 10)
  eng, params = VH.engine(VH.write_model(tmp_path, cfg, w), slots=1, pages=60, target=420, rows=32)
  t = VH.tokens(cfg, 9, 3)
  out = decode_greedy(eng, params, t, 400)
  assert_greedy(out, L.forward(cfg, w, np.concatenate([t, out])[:-1])[len(t) - 1:])
  eng.close()


def test_greedy_generation_by_every_entry_point(tmp_path, capsys):
  """MaxEngine.prefill / insert / generate (graph and eager), StepScheduler.generate and the command line give the restatement's greedy tokens."""
  cfg = LH.mixed_model()
  w = LH.random_weights(cfg, 11)
  path = VH.write_model(tmp_path, cfg, w)
  prompts = {i: VH.tokens(cfg, (13, 30, 4, 21, 8)[i], 60 + i) for i in range(5)}
  N = 20
  eng, params = VH.engine(path, slots=3)
  eager, eparams = VH.engine(path, slots=3, ixt_use_hip_graph=False)
  by_steps = VH.scheduler(eng).generate({k: v.tolist() for k, v in prompts.items()}, N, portion=6)
  for i, p in prompts.items():
    out = np.array(by_steps[i])
    assert_greedy(out, L.forward(cfg, w, np.concatenate([p, out])[:-1])[len(p) - 1:])
    assert (decode_greedy(eng, params, p, N, slot=i % 3) == out).all()
    assert (decode_greedy(eager, eparams, p, N, slot=(i + 1) % 3) == out).all()
  eng.close()
  eager.close()
  decode = importlib.import_module("maxtext-indextts2_amd.decode")
  decode.main(["decode", H.BASE_YML, f"ixt_model_dir={path}", "dtype=float32", "attention=paged", "scan_layers=false", "per_device_batch_size=1", "max_prefill_predict_length=32",
               "max_target_length=40", "pagedattn_tokens_per_page=8", "pagedattn_num_pages=16", "ixt_prompt_tokens=" + ",".join(map(str, prompts[0])),
               "autoregressive_decode_assert=" + ",".join(map(str, by_steps[0][:8]))])
  assert str(by_steps[0][0]) in capsys.readouterr().out


@pytest.mark.parametrize("dtype", DTYPES)
def test_graph_replays_equal_eager_steps(tmp_path, dtype):
  """Three slots decoding together: every replay of the captured step against the same step run eagerly, with other eager work in between."""
  cfg = LH.mixed_model()
  path = VH.write_model(tmp_path, cfg, LH.random_weights(cfg, 12))
  engs = [VH.engine(path, dtype=dtype, slots=3, pages=30, ixt_use_hip_graph=g) for g in (True, False)]
  states = []
  for eng, params in engs:
    st = eng.init_decode_state(materialize_logits=True)
    for i, n in enumerate((17, 3, 25)):
      padded = np.zeros(eng.max_prefill_length, np.int32)
      padded[:n] = VH.tokens(cfg, n, 70 + i)
      prefix, _ = eng.prefill(params=params, padded_tokens=padded, true_length=n, slot=i)
      st = eng.insert(prefix, st, i)
    states.append(st)
  for k in range(25):
    data = []
    for j, (eng, params) in enumerate(engs):
      states[j], r = eng.generate(params, states[j])
      data.append((r.data.cpu().numpy(), states[j]["logits"].cpu().numpy().copy()))
    assert (data[0][0] == data[1][0]).all() and np.array_equal(data[0][1], data[1][1]), k
    if k == 10:
      torch.cuda.synchronize()
      torch.zeros(1 << 20, device="cuda").add_(1)
  for eng, _ in engs:
    eng.close()


def test_packed_prefill_and_inserts_carry_the_pages(tmp_path):
  """prefill_concat + insert_partial (page lists move), bulk_insert (keys and values are copied)."""
  cfg = LH.mixed_model()
  w = LH.random_weights(cfg, 13)
  eng, params = VH.engine(VH.write_model(tmp_path, cfg, w), slots=4, pages=40, ixt_staging_groups=3, ixt_max_packed_rows=96)
  lens = [21, 6, 30]
  toks = [VH.tokens(cfg, n, 80 + n) for n in lens]
  cache, res, _ = eng.prefill_concat(params=params, padded_tokens=np.concatenate(toks), decoder_positions=np.concatenate([np.arange(n) for n in lens]), decoder_segment_ids=None,
                                     start_pos=np.cumsum([0] + lens[:-1]), true_lengths=lens, num_prompts=3)
  st = eng.insert_partial(res, eng.init_decode_state(), cache, [2, 0, 3], num_prompts=3)
  outs = {i: [int(res["tokens"][i].reshape(-1)[0])] for i in range(3)}
  for _ in range(12):
    st, r = eng.generate(params, st)
    for i, slot in enumerate((2, 0, 3)):
      outs[i].append(int(r.data[slot, 0]))
  for i in range(3):
    assert_greedy(outs[i], L.forward(cfg, w, np.concatenate([toks[i], outs[i]])[:-1])[lens[i] - 1:])
  for s in range(4):
    eng.release_pages(s)
  padded = np.zeros(eng.max_prefill_length, np.int32)
  padded[:21] = toks[0]
  prefix, _ = eng.prefill(params=params, padded_tokens=padded, true_length=21, slot=1)
  st = eng.bulk_insert(prefix, eng.init_decode_state(), [1, 3, 0])
  for k in range(1, 10):
    st, r = eng.generate(params, st)
    assert [int(r.data[s, 0]) for s in (1, 3, 0)] == [outs[0][k]] * 3
  eng.close()


def decode_all(cfg, w, eng, params, lens, steps, seed):
  """All slots decode together; -> (logits of every step [steps, slots, vocab], what the restatement gives for the same tokens)."""
  B = len(lens)
  st = eng.init_decode_state(materialize_logits=True)
  seqs, got = [], []
  for i, n in enumerate(lens):
    padded = np.zeros(eng.max_prefill_length, np.int32)
    padded[:n] = VH.tokens(cfg, n, seed + i)
    prefix, first = eng.prefill(params=params, padded_tokens=padded, true_length=n, slot=i)
    st = eng.insert(prefix, st, i)
    seqs.append(list(padded[:n]) + [int(first.data[0, 0])])
  for _ in range(steps):
    st, r = eng.generate(params, st)
    got.append(st["logits"].cpu().numpy().reshape(B, -1).copy())
    for i, tok in enumerate(r.data.cpu().numpy()[:, 0]):
      seqs[i].append(int(tok))
  return np.stack(got), np.stack([L.forward(cfg, w, s[:-1])[-steps:] for s in seqs], axis=1)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(MIXERS))
def test_decode_step_alone(tmp_path, name, dtype):
  """The decode step's own attention (queries, key and value straight from the projection) at every size: positions around page and tile borders."""
  cfg = LH.model([LH.with_mlp(MIXERS[name], None)])
  w = LH.random_weights(cfg, 2)
  eng, params = VH.engine(VH.write_model(tmp_path, cfg, w), dtype=dtype, slots=3, pages=40, target=90, rows=80)
  got, want = decode_all(cfg, w, eng, params, (1, 61, 36), 9, 300)
  for i in range(3):
    LH.check(got[:, i], want[:, i], dtype, (name, i))
  eng.close()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("slots", [40, 130])
def test_many_slots_decode_together(tmp_path, slots, dtype):
  """Sequences of unequal length: the decode step's forms for some tens and for more than 128 rows."""
  cfg = LH.mixed_model()
  w = LH.random_weights(cfg, 5)
  eng, params = VH.engine(VH.write_model(tmp_path, cfg, w), dtype=dtype, slots=slots, pages=5 * slots, target=40, rows=32)
  got, want = decode_all(cfg, w, eng, params, [1 + (7 * i) % 30 for i in range(slots)], 4, 200)
  for k in range(4):
    LH.check(got[k], want[k], dtype, k)
  eng.close()


def test_chunked_prefill_prompt_logp_and_sampling_ranges(tmp_path):
  cfg = LH.mixed_model()
  w = LH.random_weights(cfg, 14)
  eng, params = VH.engine(VH.write_model(tmp_path, cfg, w), slots=2)
  t = VH.tokens(cfg, 50, 90)
  want = L.forward(cfg, w, t)
  logp = want - np.log(np.exp(want - want.max(axis=1, keepdims=True)).sum(axis=1, keepdims=True)) - want.max(axis=1, keepdims=True)
  prefix, _ = eng.prefill(params=params, padded_tokens=t[:30], true_length=30, slot=1, return_prompt_logp=True)
  assert np.abs(prefix["prompt_logp"].cpu().numpy()[0] - logp[np.arange(30), t[:30]]).max() < 1e-3
  old = H.maxengine_module().ExistingPrefix(cache=prefix["cache"], common_prefix_tokens=t[:30])
  nxt, _ = eng.prefill(params=params, existing_prefix=old, padded_tokens=t[30:], true_length=20, slot=1)
  LH.check(nxt["logits"].cpu().numpy().reshape(1, -1), want[49:50], "float32")
  with pytest.raises(ValueError, match="state"):        # the state stands at 50 tokens; it cannot go back to 30
    eng.prefill(params=params, existing_prefix=old, padded_tokens=t[30:], true_length=20, slot=1)
  eng.set_sampling_ranges([(3, 40), (100, 150)])
  _, tok = VH.scheduler(eng).step([("r", t, [49])])
  allowed = np.full_like(want[49], -np.inf)
  for a, b in ((3, 40), (100, 150)):
    allowed[a:b] = want[49, a:b]
  assert tok.cpu().tolist() == [int(allowed.argmax())]
  eng.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_trace_runner(tmp_path, dtype):
  """The trace program, in this process: steps in, one logits file per step out."""
  cfg = LH.mixed_model()
  w = LH.random_weights(cfg, 5)
  path = VH.write_model(tmp_path / "m", cfg, w)
  a, b = VH.tokens(cfg, 70, 1), VH.tokens(cfg, 12, 2)
  steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:64].tolist(), "want": [0, 63]}], "end": []},
           {"step": 1, "entries": [{"id": "b", "tokens": b[:11].tolist(), "want": []}], "end": []},
           {"step": 2, "entries": [{"id": "a", "tokens": a[64:].tolist(), "want": [5]}, {"id": "b", "tokens": b[11:].tolist(), "want": [0]}], "end": ["a", "b"]},
           {"step": 3, "entries": [{"id": "a", "tokens": b.tolist(), "want": [11]}], "end": ["a"]}]
  run = importlib.import_module("maxtext-indextts2_amd.trace_run")
  stdin, out = sys.stdin, io.StringIO()
  try:
    sys.stdin = io.StringIO("\n".join(map(json.dumps, steps)) + "\n")
    with contextlib.redirect_stdout(out):
      assert run.main(["--model", path, "--dtype", dtype, "--out", str(tmp_path / "o"), "--max-tokens", "192"]) == 0
  finally:
    sys.stdin = stdin
  assert [l for l in out.getvalue().split("\n") if l.startswith("done")] == [f"done {i}" for i in range(4)]
  load = lambda i: np.fromfile(tmp_path / "o" / f"{i}.f32", "<f4").reshape(-1, cfg["vocab"])
  wa, wb = L.forward(cfg, w, a), L.forward(cfg, w, b)
  assert not (tmp_path / "o" / "1.f32").exists()
  LH.check(load(0), wa[[0, 63]], dtype)
  LH.check(load(2), np.stack([wa[69], wb[11]]), dtype)
  LH.check(load(3), wb[11:12], dtype)
