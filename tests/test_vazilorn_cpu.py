"""Vazilorn without a GPU: the folder reader and its registry, synthetic parameters, and properties of the plain restatement (vazilorn_ref) that the GPU
tests rest on -- also that a planted mistake would show in them."""
import importlib
import json

import numpy as np
import pytest

import helpers as H
import vazilorn_helpers as ZH
import vazilorn_ref as Z
import vilepel_helpers as VH

arch = importlib.import_module("maxtext-indextts2_amd.architectures")


def test_reader_takes_every_size_from_the_folder(tmp_path):
  cfg = ZH.mixed_model()
  w = ZH.random_weights(cfg)
  c = VH.config(VH.write_model(tmp_path, cfg, w))
  assert (c.vocab_size, c.emb_dim, c.normalization_layer_epsilon, c.embedding_scale, c.decoder_block) == (203, 88, 3e-5, 1.0, "hybrid")
  assert (c.hybrid_norm_kind, c.hybrid_norm_places) == (arch.NORM_TANH, arch.NORM_BEFORE | arch.NORM_AFTER)
  l = c.hybrid_layers
  assert all((x.mixer, x.weights_of, x.qk_norm, x.sink) == (arch.MIX_ATTENTION, -1, 1, 1) for x in l)
  assert [x.ffn for x in l] == [1, 2, 0, 2, 1] and [x.glu for x in l if x.ffn] == [arch.GLU_GELU_TANH, arch.GLU_SILU, arch.GLU_SILU, arch.GLU_GELU_TANH]
  assert (l[1].heads, l[1].kv_heads, l[1].dim, l[1].vdim, l[1].rot_dim, l[1].window, l[1].rope_base, l[1].attn_scale, l[1].rope_factor) == (5, 1, 40, 12, 6, 19, 900.0, 0.2, 0.0)
  assert (l[0].rope_factor, l[0].rope_low, l[0].rope_high, l[0].rope_original) == (4.0, 1.0, 4.0, 40.0)
  assert (l[3].experts, l[3].top, l[3].groups, l[3].groups_keep, l[3].router_scale, l[3].shared_ff, l[3].ff) == (8, 2, 4, 1, 0.6, 200, 24)
  assert (l[3].router, l[3].router_correction, l[3].router_norm) == (arch.ROUTE_SIGMOID, 1, 1)
  used = {k: v.shape for k, v in w.items() if not k.startswith("l2.norm2")}          # (a layer without feed-forward does not need its norms)
  assert arch.parameter_shapes(c) == used


def test_synthetic_parameters(tmp_path):
  with open(tmp_path / "config.json", "w", encoding="utf-8") as f:
    json.dump(ZH.mixed_model(), f)
  c = VH.config(tmp_path)
  assert c.load_parameters_path == ""
  shapes = arch.parameter_shapes(c)
  w = H.synth.synth_weights(c, 3)
  assert {k: v.shape for k, v in w.items()} == shapes
  spec = H.synth.device_tree_spec(c)
  assert {n: s for n, s, _ in spec} == shapes


def test_reader_refuses_what_it_does_not_know(tmp_path):
  cfg = ZH.mixed_model()
  z = {"embed": np.zeros((2, 2))}
  for i, (change, text) in enumerate((({"type": "other"}, "type"), ({"mlp": {"kind": "other"}}, "kind"),
                                      ({"mixer": dict(cfg["layers"][0]["mixer"], kv_heads=4)}, "heads"),
                                      ({"mixer": dict(cfg["layers"][0]["mixer"], rot={"base": 10.0, "dims": 26})}, "rotated"))):
    with pytest.raises(ValueError, match=text):
      VH.config(VH.write_model(tmp_path / str(i), dict(cfg, layers=[dict(cfg["layers"][0], **change)]), z))


# ---------------------------------------------------------------------------------------------------- the restatement
def test_rotation_against_complex_numbers_and_frequency_regimes():
  x = np.random.default_rng(0).standard_normal((5, 9))
  pos = np.arange(5.0)
  rot = {"base": 100.0, "dims": 6, "scaling": None}
  y = Z.rotate_first(x, pos, rot)
  z = (x[:, 0:6:2] + 1j * x[:, 1:6:2]) * np.exp(1j * pos[:, None] * 100.0 ** (-np.arange(0, 6, 2) / 6))
  assert np.allclose(y[:, 0:6:2] + 1j * y[:, 1:6:2], z) and (y[:, 6:] == x[:, 6:]).all()
  plain = Z.frequencies(16, 300.0, None)
  f = Z.frequencies(16, 300.0, ZH.SCALING)
  turns = ZH.SCALING["original"] * plain / (2 * np.pi)
  assert (turns > 4).any() and ((turns < 4) & (turns > 1)).any() and (turns < 1).any()
  assert np.allclose(f[turns > 4], plain[turns > 4]) and np.allclose(f[turns < 1], plain[turns < 1] / 4)
  mid = (turns < 4) & (turns > 1)
  assert (f[mid] < plain[mid]).all() and (f[mid] > plain[mid] / 4).all()


def test_sink_and_window():
  s = np.random.default_rng(1).standard_normal((6, 6))
  p = Z.sink_softmax(s, 3, 0.7)
  for i in range(6):
    j = np.arange(max(0, i - 2), i + 1)
    e = np.exp(s[i, j])
    assert np.allclose(p[i, j], e / (e.sum() + np.exp(0.7))) and np.allclose(p[i].sum(), p[i, j].sum())
  assert np.allclose(Z.sink_softmax(s, 3, -1e4).sum(axis=1), 1.0)


def test_router_rules():
  r = {"experts": 6, "top": 2, "groups": {"count": 3, "keep": 1}, "scale": 2.0}
  h = np.eye(6)[:1]
  router = np.array([[2.0], [-9.0], [1.0], [1.0], [1.9], [-9.0]]) * h      # the single best expert is not in the best pair of neighbours
  picks, weights = Z.route(h, router, np.zeros(6), r)
  assert sorted(picks[0]) == [2, 3] and np.allclose(weights[0], 1.0)
  corr = np.array([-3.0, -3.0, -5.0, -5.0, -3.0, -3.0])                     # all choice scores negative; the correction moves the choice, not the weights
  picks, weights = Z.route(h, router, corr, r)
  assert sorted(picks[0]) == [0, 1]
  s = Z.sigmoid(np.array([2.0, -9.0]))
  assert np.allclose(weights[0], 2.0 * s[[int(p) for p in picks[0]]] / s.sum())


def test_restatement_is_causal_and_windowed():
  cfg = ZH.mixed_model()
  w = ZH.random_weights(cfg, 1)
  t = VH.tokens(cfg, 40, 2)
  full = Z.forward(cfg, w, t)
  assert np.allclose(Z.forward(cfg, w, t[:23]), full[:23], atol=1e-12)
  only = ZH.model([ZH.with_mlp(ZH.attn(window=7), None)])
  wo = ZH.random_weights(only, 1)
  a = VH.tokens(only, 30, 3)
  b = a.copy()
  b[10] = (b[10] + 1) % only["vocab"]
  d = np.abs(Z.forward(only, wo, a) - Z.forward(only, wo, b)).max(axis=1)
  assert (d[10:17] > 1e-6).all() and d[17:].max() < 1e-12 and d[:10].max() < 1e-12


def _planted(cfg, w, toks, **changes):
  """The restatement with one mistake: functions of vazilorn_ref replaced for the call."""
  saved = {k: getattr(Z, k) for k in changes}
  try:
    for k, f in changes.items():
      setattr(Z, k, f)
    return Z.forward(cfg, w, toks)
  finally:
    for k, f in saved.items():
      setattr(Z, k, f)


def _silent(w, part):
  return {k: np.zeros_like(v) if part in k else v for k, v in w.items()}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_planted_mistakes_would_show(dtype):
  """Each mistake moves the logits of the model that the GPU tests run by more than their tolerance."""
  cfg = ZH.mixed_model()
  w = ZH.random_weights(cfg, 5)
  t = VH.tokens(cfg, 60, 6)
  good = Z.forward(cfg, w, t)
  sm, rot, fr, route, gu, norm, att = Z.sink_softmax, Z.rotate_first, Z.frequencies, Z.route, Z.gated_unit, Z.tanh_norm, Z.attention
  groups = lambda r, **kw: dict(r, groups=dict(r["groups"], **kw))
  mistakes = {
      "window one short": dict(sink_softmax=lambda s, n, k: sm(s, n - 1, k)),
      "window one long": dict(sink_softmax=lambda s, n, k: sm(s, n + 1, k)),
      "no sink": dict(sink_softmax=lambda s, n, k: sm(s, n, -1e4)),
      "sink counted twice": dict(sink_softmax=lambda s, n, k: sm(s, n, k + np.log(2.0))),
      "no frequency scaling": dict(frequencies=lambda d, b, s: fr(d, b, None)),
      "all features turn": dict(rotate_first=lambda x, p, r: rot(x, p, dict(r, dims=x.shape[1] // 2 * 2))),
      "heads on the wrong key head": dict(attention=lambda h, x, m, e: att(h, dict(x, k=np.roll(x["k"], m["dim"], axis=0)), m, e)),
      "no head norm weight": dict(attention=lambda h, x, m, e: att(h, dict(x, **{"k.norm": np.ones(m["dim"])}), m, e)),
      "no correction": dict(route=lambda h, r, c, m: route(h, r, 0 * c, m)),
      "no groups": dict(route=lambda h, r, c, m: route(h, r, c, groups(m, keep=m["groups"]["count"]))),
      "weights not divided": dict(route=lambda h, r, c, m: (route(h, r, c, m)[0], [Z.sigmoid(r @ h[i])[p] for i, p in enumerate(route(h, r, c, m)[0])])),
      "no shared unit": None,
      "silu for gelu": dict(gelu_tanh=Z.silu),
      "no norm offset": dict(tanh_norm=lambda x, a, v, b: norm(x, a, v, 0 * b)),
  }
  for name, change in mistakes.items():
    bad = Z.forward(cfg, _silent(w, "shared.down"), t) if change is None else _planted(cfg, w, t, **change)
    worst = np.quantile(VH.rel(bad, good)[31:], 0.9)
    print(dtype, name, worst)
    assert worst > ZH.TOL[dtype] * (1.5 if dtype == "float32" else 1.0), (name, worst)
