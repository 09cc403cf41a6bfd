"""Vilepel without a GPU: the folder reader and its registry, configuration errors, the scheduler's bookkeeping, and properties of the plain
restatement (vilepel_ref) that the GPU tests rest on -- also that a planted mistake would show in them."""
import importlib

import numpy as np
import pytest

import helpers as H
import vilepel_helpers as VH
import vilepel_ref as V

arch = importlib.import_module("maxtext-indextts2_amd.architectures")


def test_reader_takes_every_size_from_the_folder(tmp_path):
  cfg = VH.mixed_model()
  w = VH.random_weights(cfg, decay_rank=9, gate_rank=5)
  c = VH.config(VH.write_model(tmp_path, cfg, w))
  assert (c.vocab_size, c.emb_dim, c.normalization_layer_epsilon, c.embedding_scale, c.decoder_block) == (203, 88, 3e-5, 2.5, "hybrid")
  assert c.load_parameters_path == str(tmp_path / "model.safetensors")
  l = c.hybrid_layers
  assert [x.mixer for x in l] == [1, 0, 0, 0, 1, 1] and [x.weights_of for x in l] == [-1, -1, -1, 1, 0, -1] and [x.ffn for x in l] == [2, 1, 2, 1, 2, 0]
  assert (l[0].decay_rank, l[0].gate_rank, l[0].conv, l[0].kv_heads) == (9, 5, 4, 3)
  assert (l[4].decay_rank, l[4].gate_rank) == (9, 5)                   # a sharing layer's ranks come from the tensors it uses
  assert (l[2].kv_rank, l[2].rot_dim, l[2].window, l[2].rope_base, l[2].attn_scale) == (72, 6, 19, 500.0, 0.3)
  assert (l[2].experts, l[2].top, l[2].ff, l[2].glu_limit) == (7, 2, 24, 1.25)
  assert arch.parameter_shapes(c) == {k: v.shape for k, v in w.items()}


def test_reader_without_weights_and_synthetic_parameters(tmp_path):
  import json
  cfg = VH.mixed_model()
  with open(tmp_path / "config.json", "w", encoding="utf-8") as f:
    json.dump(cfg, f)
  c = VH.config(tmp_path)
  assert c.load_parameters_path == "" and c.hybrid_layers[0].decay_rank == cfg["layers"][0]["mixer"]["dim"]
  w = H.synth.synth_weights(c, 3)
  assert {k: v.shape for k, v in w.items()} == arch.parameter_shapes(c)


def test_reader_refuses_what_it_does_not_know(tmp_path):
  cfg = VH.mixed_model()
  VH.write_model(tmp_path, cfg, {"embed": np.zeros((2, 2))})
  bad = dict(cfg, architecture="Nobody")
  VH.write_model(tmp_path / "a", bad, {"embed": np.zeros((2, 2))})
  with pytest.raises(ValueError, match="not built"):
    VH.config(tmp_path / "a")
  bad = dict(cfg, layers=[dict(cfg["layers"][0], type="other")])
  VH.write_model(tmp_path / "b", bad, {"embed": np.zeros((2, 2))})
  with pytest.raises(ValueError, match="type"):
    VH.config(tmp_path / "b")
  with pytest.raises(ValueError, match="model folder"):
    VH.config(tmp_path, vocab_size=7)
  with pytest.raises(ValueError, match="model_name"):
    VH.config(tmp_path, model_name="ixt-tiny")
  with pytest.raises(ValueError, match="hybrid"):
    H.make_config(decoder_block="hybrid")


class _FakeEngine:
  max_concurrent_decodes = 2

  def __init__(self):
    self.calls, self.released = [], []

  def step(self, batch, want_logits=True):
    self.calls.append(batch)
    return None, [sum(b[2]) % 97 for b in batch for _ in b[3]]

  def release_pages(self, slot):
    self.released.append(slot)


def test_scheduler_bookkeeping():
  eng = _FakeEngine()
  s = VH.scheduler(eng)
  s.step([("a", [1, 2, 3], [2]), ("b", [4], [])])
  s.step([("b", [5, 6], [0])])                       # a is left out of a step and goes on later
  s.step([("a", [7], [0])])
  assert [[(b[1], b[2]) for b in c] for c in eng.calls] == [[(0, [1, 2, 3]), (0, [4])], [(1, [5, 6])], [(3, [7])]]
  with pytest.raises(ValueError, match="no free slot"):
    s.step([("c", [1], [])])
  slot = eng.calls[0][0][0]
  s.release("a")
  assert eng.released == [slot]
  s.step([("c", [1], [])])
  assert eng.calls[-1][0][0] == slot and eng.calls[-1][0][1] == 0      # the slot again, from its start
  with pytest.raises(ValueError, match="two entries"):
    s.step([("c", [1], []), ("c", [2], [])])
  with pytest.raises(ValueError, match="not live"):
    s.release("a")


def test_scheduler_generate_mixes_portions_and_tokens():
  eng = _FakeEngine()
  out = VH.scheduler(eng).generate({"a": [1, 2, 3, 4, 5], "b": [6], "c": [7, 8]}, 3, portion=2)
  assert {k: len(v) for k, v in out.items()} == {"a": 3, "b": 3, "c": 3}
  assert out["b"][0] == 6 and out["b"][1] == 6                         # the fake repeats the sum of what it is given
  assert any(len({len(b[2]) for b in c}) > 1 for c in eng.calls)       # portions beside single tokens
  assert sorted(eng.released) == [0, 0, 1] or sorted(eng.released) == [0, 1, 1]


def test_restatement_is_causal_and_windowed():
  cfg = VH.mixed_model()
  w = VH.random_weights(cfg, 1)
  t = VH.tokens(cfg, 40, 2)
  full = V.forward(cfg, w, t)
  assert np.allclose(V.forward(cfg, w, t[:23]), full[:23], atol=1e-12)
  only = VH.model([VH.with_mlp(VH.latent(window=7), None)])
  wo = VH.random_weights(only, 1)
  a, b = VH.tokens(only, 30, 3), VH.tokens(only, 30, 3)
  b[10] = (b[10] + 1) % only["vocab"]
  d = np.abs(V.forward(only, wo, a) - V.forward(only, wo, b)).max(axis=1)
  assert (d[10:17] > 1e-6).all() and d[17:].max() < 1e-12 and d[:10].max() < 1e-12


def test_rotation_and_delta_rule_against_closed_forms():
  x = np.random.default_rng(0).standard_normal((5, 6))
  pos = np.arange(5.0)
  z = x[:, 0::2] + 1j * x[:, 1::2]
  want = z * np.exp(1j * pos[:, None] * 100.0 ** (-np.arange(0, 6, 2) / 6))
  got = V.rotate_pairs(x, pos, 100.0)
  assert np.allclose(got[:, 0::2] + 1j * got[:, 1::2], want)
  # no decay, beta 1, orthonormal keys: the state returns exactly what was written
  k = np.eye(4)
  v = np.random.default_rng(1).standard_normal((4, 3))
  o = V.delta_rule(k, k, v, np.ones((4, 4)), np.ones(4))
  assert np.allclose(o, v)
  again = V.delta_rule(np.vstack([k, k[1:2]]), np.vstack([k, k[2:3]]), np.vstack([v, v[:1]]), np.ones((5, 4)), np.array([1, 1, 1, 1, 0.0]))
  assert np.allclose(again[4], v[1])


def _planted(cfg, w, toks, **changes):
  """The restatement with one mistake: functions of vilepel_ref replaced for the call."""
  saved = {k: getattr(V, k) for k in changes}
  try:
    for k, f in changes.items():
      setattr(V, k, f)
    return V.forward(cfg, w, toks)
  finally:
    for k, f in saved.items():
      setattr(V, k, f)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_planted_mistakes_would_show(dtype):
  """Each mistake moves the logits of the model that the GPU tests run by more than their tolerance."""
  cfg = VH.mixed_model()
  w = VH.random_weights(cfg, 5)
  t = VH.tokens(cfg, 60, 6)
  good = V.forward(cfg, w, t)
  ws, conv, rot, glu, route, unit, dr = V.window_softmax, V.short_conv, V.rotate_pairs, V.clamped_glu, V.route, V.unit, V.delta_rule
  mistakes = {
      "window one short": dict(window_softmax=lambda s, n: ws(s, n - 1)),
      "window one long": dict(window_softmax=lambda s, n: ws(s, n + 1)),
      "taps reversed": dict(short_conv=lambda x, k: conv(x, k[:, ::-1])),
      "positions off by one key": dict(rotate_pairs=lambda x, p, b: rot(x, p * 1.02, b)),
      "no clamp": dict(clamped_glu=lambda h, a, b, c, limit: glu(h, a, b, c, 1e9)),
      # (renormalizing the router's weights scales a row's whole output, which the norm behind it takes out again: no model-level test can see it)
      "router weights ignored": dict(route=lambda h, r, k: (route(h, r, k)[0], np.ones_like(route(h, r, k)[1]))),
      "keys not unit": dict(unit=lambda x: x),
      "state lost at 30": dict(delta_rule=lambda q, k, v, g, b: np.concatenate([dr(q[:30], k[:30], v[:30], g[:30], b[:30]), dr(q[30:], k[30:], v[30:], g[30:], b[30:])])),
      "read before write": dict(delta_rule=lambda q, k, v, g, b: dr(q, k, v, g, b) - b[:, None] * np.sum(q * k, axis=1, keepdims=True) * v),
  }
  for name, change in mistakes.items():
    r = VH.rel(_planted(cfg, w, t, **change), good)
    worst = np.quantile(r[31:], 0.9)
    print(dtype, name, worst)
    assert worst > VH.TOL[dtype] * (1.5 if dtype == "float32" else 1.0), (name, worst)
