"""Suzulix without a GPU: the folder reader and its registry, synthetic parameters, and properties of the plain restatement (suzulix_ref) that the GPU
tests rest on -- also that a planted mistake would show in them."""
import importlib
import json

import numpy as np
import pytest

import helpers as H
import suzulix_helpers as SH
import suzulix_ref as S
import vilepel_helpers as VH

arch = importlib.import_module("maxtext-indextts2_amd.architectures")


def test_reader_takes_every_size_from_the_folder(tmp_path):
  cfg = SH.mixed_model()
  w = SH.random_weights(cfg)
  c = VH.config(VH.write_model(tmp_path, cfg, w))
  assert (c.vocab_size, c.emb_dim, c.normalization_layer_epsilon, c.embedding_scale, c.decoder_block, c.logit_scale, c.hybrid_streams) == (203, 88, 3e-5, 2.5, "hybrid", 1.5, 3)
  assert (c.hybrid_norm_kind, c.hybrid_norm_places, c.logits_via_embedding, c.num_decoder_layers) == (arch.NORM_LAYER, arch.NORM_BEFORE, True, 9)
  l = c.hybrid_layers
  assert [x.number for x in l] == [0, 1, 2, 3, 1, 2, 3, 4, 5] == S.layer_runs(cfg)
  assert [x.weights_of for x in l] == [-1] * 4 + [1, 2, 3, -1, -1]
  assert [x.mixer for x in l] == [arch.MIX_LATENT_ATTENTION, arch.MIX_RETENTION, arch.MIX_ATTENTION, arch.MIX_ATTENTION, arch.MIX_RETENTION, arch.MIX_ATTENTION, arch.MIX_ATTENTION,
                                  arch.MIX_RETENTION, arch.MIX_LATENT_ATTENTION]
  assert (l[8].heads, l[8].dim, l[8].rot_dim, l[8].vdim, l[8].kv_rank, l[8].q_rank, l[8].rope_base, l[8].attn_scale, l[8].rope_pairs, l[8].out_gate) == (5, 12, 6, 16, 72, 20, 90.0, 0.3, 1, 1)
  assert (l[3].heads, l[3].kv_heads, l[3].dim, l[3].vdim, l[3].rot_dim, l[3].softcap, l[3].map_diff, l[3].maps, l[3].rope_pairs, l[3].out_gate) == (4, 1, 30, 24, 30, 15.0, 0.6, 2, 0, 1)
  assert (l[7].heads, l[7].dim, l[7].vdim, l[7].rot_dim, l[7].decay, l[7].rope_pairs) == (2, 34, 18, 34, (0.5, 0.9990234375), 1)
  assert (l[3].experts, l[3].top, l[3].ff, l[3].shared_ff, l[3].shared_gate, l[3].router, l[3].router_bias, l[3].glu) == (4, 1, 16, 140, 1, arch.ROUTE_CHOSEN, 1, arch.ACT_RELU2)
  assert (l[1].shared_ff, l[1].shared_gate, l[2].ffn) == (0, 0, arch.FFN_NONE)
  assert arch.parameter_shapes(c) == {k: v.shape for k, v in w.items()}


def test_loops(tmp_path):
  layers = [SH.with_mlp(SH.attn(), None)] * 3
  for i, (loop, want) in enumerate(((None, [0, 1, 2]), ({"start": 0, "stop": 3, "times": 1}, [0, 1, 2]), ({"start": 2, "stop": 3, "times": 3}, [0, 1, 2, 2, 2]),
                                    ({"start": 0, "stop": 1, "times": 2}, [0, 0, 1, 2]), ({"start": 0, "stop": 2, "times": 2}, [0, 1, 0, 1, 2]))):
    cfg = SH.model(layers, loop=loop)
    c = VH.config(VH.write_model(tmp_path / str(i), cfg, {"embed": np.zeros((2, 2))}))
    assert [x.number for x in c.hybrid_layers] == want == S.layer_runs(cfg)
  for loop in ({"start": 2, "stop": 4, "times": 2}, {"start": 2, "stop": 1, "times": 2}, {"start": 0, "stop": 2, "times": 0}):
    with pytest.raises(ValueError, match="loop"):
      VH.config(VH.write_model(tmp_path / "x", SH.model(layers, loop=loop), {"embed": np.zeros((2, 2))}))


def test_synthetic_parameters(tmp_path):
  with open(tmp_path / "config.json", "w", encoding="utf-8") as f:
    json.dump(SH.mixed_model(), f)
  c = VH.config(tmp_path)
  assert c.load_parameters_path == ""
  shapes = arch.parameter_shapes(c)
  assert "head" not in shapes
  w = H.synth.synth_weights(c, 3)
  assert {k: v.shape for k, v in w.items()} == shapes
  assert {n: s for n, s, _ in H.synth.device_tree_spec(c)} == shapes


def test_reader_refuses_what_it_does_not_know(tmp_path):
  cfg = SH.mixed_model()
  z = {"embed": np.zeros((2, 2))}
  m = [dict(l["mixer"]) for l in cfg["layers"]]
  for i, (at, change, text) in enumerate(((0, {"type": "other"}, "type"), (0, {"mlp": {"kind": "dense"}}, "kind"), (0, {"mixer": dict(m[0], rot={"base": 9.0, "dims": 4})}, "rot_dim"),
                                          (2, {"mixer": dict(m[2], kv_heads=4)}, "heads"), (2, {"mixer": dict(m[2], rot={"base": 9.0, "dims": 20})}, "rotated"),
                                          (1, {"mixer": dict(m[1], decay=[0.5])}, "decays"))):
    layers = list(cfg["layers"])
    layers[at] = dict(layers[at], **change)
    with pytest.raises(ValueError, match=text):
      VH.config(VH.write_model(tmp_path / str(i), dict(cfg, layers=layers), z))


# ---------------------------------------------------------------------------------------------------- the restatement
def test_rotations_against_complex_numbers():
  x = np.random.default_rng(0).standard_normal((5, 9))
  pos, rot = np.arange(5.0), {"base": 100.0, "dims": 6}
  turn = np.exp(1j * pos[:, None] * 100.0 ** (-np.arange(0, 6, 2) / 6))
  y = S.rotate_neighbours(x, pos, rot)
  assert np.allclose(y[:, 0:6:2] + 1j * y[:, 1:6:2], (x[:, 0:6:2] + 1j * x[:, 1:6:2]) * turn) and (y[:, 6:] == x[:, 6:]).all()
  y = S.rotate_halves(x, pos, rot)
  assert np.allclose(y[:, :3] + 1j * y[:, 3:6], (x[:, :3] + 1j * x[:, 3:6]) * turn) and (y[:, 6:] == x[:, 6:]).all()


def test_retention_equals_its_sum_over_the_past():
  rng = np.random.default_rng(1)
  q, k, v = rng.standard_normal((7, 4)), rng.standard_normal((7, 4)), rng.standard_normal((7, 3))
  o = S.retention_states(q, k, v, 0.7)
  for t in range(7):
    assert np.allclose(o[t], sum(0.7 ** (t - j) * (q[t] @ k[j]) * v[j] for j in range(t + 1)))


def test_streams_with_neutral_numbers_are_one_residual_sum():
  rng = np.random.default_rng(2)
  x, y = rng.standard_normal((5, 1, 6)).repeat(3, axis=1), rng.standard_normal((5, 6))
  w = {"in": np.full(3, 1 / 3), "out": np.ones(3), "mix": np.eye(3)}
  assert np.allclose(S.gather_streams(x, w), x[:, 0]) and np.allclose(S.spread_streams(x, y, w), (x[:, 0] + y)[:, None])
  w["mix"] = np.zeros((3, 3))
  w["mix"][0, 2] = 1.0                                     # from the first to the last
  z = S.spread_streams(rng.standard_normal((5, 3, 6)), 0 * y, w)
  assert (z[:, :2] == 0).all() and (z[:, 2] != 0).all()


def test_router_weights():
  h, router = np.eye(4)[:1], np.array([[1.0, 0, 0, 0], [3.0, 0, 0, 0], [-2.0, 0, 0, 0]])
  picks, weights = S.route(h, router, np.array([0.0, 0.0, 4.5]), 2)
  assert list(picks[0]) == [1, 2] and np.allclose(weights[0], np.exp([3.0, 2.5]) / np.exp([3.0, 2.5]).sum())


def test_restatement_is_causal():
  cfg = SH.mixed_model()
  w = SH.random_weights(cfg, 1)
  t = VH.tokens(cfg, 40, 2)
  assert np.allclose(S.forward(cfg, w, t[:23]), S.forward(cfg, w, t)[:23], atol=1e-10)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_planted_mistakes_would_show(dtype, monkeypatch):
  """Each mistake moves the logits of the model that the GPU tests run by more than their tolerance."""
  cfg = SH.mixed_model()
  w = SH.random_weights(cfg, 5)
  t = VH.tokens(cfg, 60, 6)
  good = S.forward(cfg, w, t)
  ret, gather, spread, lat, dif = S.retention_states, S.gather_streams, S.spread_streams, S.latent_attention, S.differential_attention
  zero = lambda *parts: {k: np.zeros_like(v) if any(p in k for p in parts) else v for k, v in w.items()}
  ones = lambda part: {k: np.ones_like(v) if k.endswith(part) else v for k, v in w.items()}

  def first_key_lost(s):
    s = s.copy()
    s[1:, 0] = -np.inf
    return soft(s)

  soft = S.causal_softmax
  mistakes = {
      "first key not seen": dict(causal_softmax=first_key_lost),
      "neighbours for halves": dict(rotate_halves=S.rotate_neighbours), "halves for neighbours": dict(rotate_neighbours=S.rotate_halves),
      "all features turn": dict(rotate_neighbours=lambda x, p, r, f=S.rotate_neighbours: f(x, p, dict(r, dims=x.shape[1] // 2 * 2))),
      "no soft cap": dict(capped=lambda s, c: s), "one map": dict(mixing_factor=lambda u, d: 0.0), "lambda is diff": dict(mixing_factor=lambda u, d: d),
      "no attention gate": {"MIXERS": dict(S.MIXERS, attention=lambda h, u, m, e: dif(h, dict(u, g=0 * u["g"]), m, e))},
      "heads on the wrong key head": {"MIXERS": dict(S.MIXERS, attention=lambda h, u, m, e: dif(h, dict(u, k=np.roll(u["k"], 2 * m["dim"], axis=0)), m, e))},
      "maps swapped": {"MIXERS": dict(S.MIXERS, attention=lambda h, u, m, e: dif(h, dict(u, k=np.roll(u["k"], m["dim"], axis=0), q=np.roll(u["q"], m["dim"], axis=0)), m, e))},
      "no latent gate": {"MIXERS": dict(S.MIXERS, latent_attention=lambda h, u, m, e: lat(h, dict(u, g=0 * u["g"]), m, e))},
      "read before written": dict(retention_states=lambda q, k, v, d: ret(q, k, v, d) - (q * k).sum(1, keepdims=True) * v), "state lost": dict(retention_states=lambda q, k, v, d: (q * k).sum(1, keepdims=True) * v),
      "decays swapped": {"MIXERS": dict(S.MIXERS, retention=lambda h, u, m, e, f=S.retention: f(h, u, dict(m, decay=m["decay"][::-1]), e))},
      "mix transposed": dict(spread_streams=lambda x, y, u: spread(x, y, dict(u, mix=u["mix"].T))), "streams not mixed": dict(spread_streams=lambda x, y, u: spread(x, y, dict(u, mix=np.eye(3)))),
      "streams averaged": dict(gather_streams=lambda x, u: x.mean(axis=1)),
      "weights over all experts": dict(route=lambda h, r, b, n, f=S.route: (f(h, r, b, n)[0], np.take_along_axis(f(h, r, b, r.shape[0])[1], np.argsort(np.argsort(-(h @ r.T + b), 1, kind="stable"), 1)[
          np.arange(len(h))[:, None], f(h, r, b, n)[0]], 1))),
      "no router bias": dict(route=lambda h, r, b, n, f=S.route: f(h, r, 0 * b, n)), "relu for its square": dict(square_unit=lambda h, u, d: S.linear(d, np.maximum(S.linear(u, h), 0))),
      "no shared unit": zero("shared.down"), "no shared gate": zero("shared.sg"), "no query norm weight": ones("dq.norm"), "no latent norm weight": ones("dkv.norm"),
      "no norm offset": zero("norm1.b", "norm2.b"),
      "no loop": dict(layer_runs=lambda c: list(range(len(c["layers"])))),
      "loop layer by layer": dict(layer_runs=lambda c: [0, 1, 1, 2, 2, 3, 3, 4, 5]),
  }
  for name, change in mistakes.items():
    with monkeypatch.context() as mp:
      if "embed" in change:
        bad = S.forward(cfg, change, t)
      else:
        for k, f in change.items():
          mp.setattr(S, k, f)
        bad = S.forward(cfg, w, t)
    worst = np.quantile(SH.rel(bad, good)[5:], 0.9)
    print(dtype, name, worst)
    assert worst > SH.TOL[dtype] * (1.5 if dtype == "float32" else 1.0), (name, worst)
