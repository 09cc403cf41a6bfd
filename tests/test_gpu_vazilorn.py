"""Vazilorn on the GPU against the plain float64 restatement (vazilorn_ref): every mechanism alone at many sizes, then the cache, the batch and the
engine's entry points.  float32 is held to rounding of f32 sums, bfloat16 to rounding of its operands (vazilorn_helpers.TOL)."""
import contextlib
import ctypes
import importlib
import io
import json
import sys

import numpy as np
import pytest
import torch

import helpers as H
import vazilorn_helpers as ZH
import vazilorn_ref as Z
import vilepel_helpers as VH

pytestmark = pytest.mark.gpu
DTYPES = ["float32", "bfloat16"]


def one_layer(tmp_path, layer, dtype, n=50, seed=0, portions=(), alter=None, outliers=False, **kw):
  """Residual stream behind one layer for a prompt (and for the same tokens in portions) against the restatement."""
  cfg = ZH.model([layer])
  w = ZH.random_weights(cfg, seed)
  if alter is not None:
    alter(w)
    w = ZH.rounded(w)
  toks = VH.tokens(cfg, n, seed + 1)
  taps = []
  Z.forward(cfg, w, toks, taps)
  eng, _ = VH.engine(VH.write_model(tmp_path, cfg, w), dtype=dtype, **kw)
  for cuts in ((n,),) + tuple(portions):
    s, got, at, i = VH.scheduler(eng), [], 0, 0
    while at < n:
      m = min(cuts[min(i, len(cuts) - 1)], n - at)
      tap = torch.zeros(m * cfg["width"], device="cuda")
      H.lib.check(eng.lib.ixt_set_residual_tap(eng._ctx, ctypes.c_void_p(tap.data_ptr()), tap.numel()))
      s.step([("r", toks[at:at + m], [])])
      got.append(tap.cpu().numpy().reshape(m, -1))
      at, i = at + m, i + 1
    s.release("r")
    r = VH.rel(np.concatenate(got), taps[0])
    if dtype == "float32":
      assert r.max() < 1e-5, (cuts, int(r.argmax()), r.max())
    else:                                           # (a close choice of experts may turn over with rounding)
      assert np.quantile(r, 0.9) < 0.015 and (r.max() < 0.03 or outliers), (cuts, int(r.argmax()), np.quantile(r, 0.9), r.max())
  eng.close()


ATTENTIONS = {
    "one head": ZH.attn(heads=1, kv_heads=1, dim=8, vdim=8, window=4, dims=8),
    "odd sizes": ZH.attn(heads=3, kv_heads=3, dim=23, vdim=17, window=11, dims=10),
    "window 1": ZH.attn(heads=2, kv_heads=1, window=1),
    "window past the end": ZH.attn(heads=6, kv_heads=2, dim=32, vdim=32, window=1000, dims=32),
    "nothing turns": ZH.attn(heads=2, kv_heads=2, dims=0, scaling=None),
    "one pair turns": ZH.attn(heads=4, kv_heads=2, dims=2, window=30),
    "many heads on one": ZH.attn(heads=20, kv_heads=1, dim=12, vdim=12, window=33, dims=12),
    "more heads than a tile": ZH.attn(heads=70, kv_heads=1, dim=8, vdim=4, window=17, dims=4),
    "keys wider": ZH.attn(heads=4, kv_heads=2, dim=120, vdim=60, window=40, dims=64),
    "values wider": ZH.attn(heads=4, kv_heads=2, dim=50, vdim=110, window=40, dims=50),
    "64": ZH.attn(heads=4, kv_heads=4, dim=64, vdim=64, window=66, dims=64),
    "90": ZH.attn(heads=6, kv_heads=3, dim=90, vdim=84, window=65, dims=90),
    "128": ZH.attn(heads=4, kv_heads=1, dim=128, vdim=128, window=64, dims=64),
    "192 and 128": ZH.attn(heads=2, kv_heads=2, dim=192, vdim=128, window=31, dims=64),
    "180 and 150": ZH.attn(heads=2, kv_heads=1, dim=180, vdim=150, window=31, dims=180),
    "256": ZH.attn(heads=2, kv_heads=1, dim=256, vdim=250, window=31, dims=64),
    "beyond the tiles": ZH.attn(heads=2, kv_heads=1, dim=270, vdim=300, window=31, dims=64),
}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(ATTENTIONS))
def test_attention_alone(tmp_path, name, dtype):
  one_layer(tmp_path, ZH.with_mlp(ATTENTIONS[name], None), dtype, n=75, portions=((1,), (33, 2), (7, 1, 40)))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("level", [-30.0, 9.0])
def test_sinks_from_absent_to_dominant(tmp_path, level, dtype):
  def sinks(w):
    w["l0.mix.sink"] += level
  one_layer(tmp_path, ZH.with_mlp(ZH.attn(window=70), None), dtype, n=75, portions=((1,), (40, 5)), alter=sinks)


@pytest.mark.parametrize("dtype", DTYPES)
def test_tanh_norm_from_linear_to_saturated(tmp_path, dtype):
  """Slopes small, large and negative in front and behind."""
  for i, (before, after) in enumerate(((0.02, 40.0), (6.0, 0.05), (-0.7, -3.0))):
    def slopes(w, before=before, after=after):
      for n in ("norm1", "norm2"):
        w[f"l0.{n}.alpha"], w[f"l0.{n}b.alpha"] = np.array(before), np.array(after)
    # (a slope of 40 behind a sublayer multiplies what rounding has left in its output)
    if dtype == "float32" or after < 10:
      one_layer(tmp_path / str(i), ZH.with_mlp(ZH.attn(), ZH.dense()), dtype, n=40, portions=((1,),), alter=slopes, outliers=True)


MLPS = {"dense": ZH.dense(), "dense, wide": ZH.dense(300), "moe": ZH.moe(), "one group": ZH.moe(groups=1, keep=1), "groups of one": ZH.moe(experts=7, groups=7, keep=4, top=3),
        "one of many": ZH.moe(ff=16, experts=72, top=1, groups=8, keep=3), "all": ZH.moe(ff=130, experts=4, top=4, groups=2, keep=2), "one expert": ZH.moe(experts=1, top=1, groups=1, keep=1),
        "shared unit in parts": ZH.moe(ff=20, shared=390), "shared unit of one": ZH.moe(ff=140, shared=1)}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(MLPS))
def test_feed_forwards(tmp_path, name, dtype):
  one_layer(tmp_path, ZH.with_mlp(ZH.attn(), MLPS[name]), dtype, n=70, portions=((1,), (9, 61)), outliers=True)


def test_negative_choice_scores(tmp_path):
  """Corrections that push every choice score below zero: closed groups must stay closed."""
  def low(w):
    w["l0.mlp.correction"] -= 4.0
  one_layer(tmp_path, ZH.with_mlp(ZH.attn(), ZH.moe(groups=3, keep=1, top=2)), "float32", n=60, portions=((1,),), alter=low)


@pytest.mark.parametrize("dtype", DTYPES)
def test_many_rows_take_the_prompt_kernels(tmp_path, dtype):
  """300 rows in one pass: the ring GEMMs, tall attention tiles and 128-row expert groups."""
  for i, layer in enumerate((ZH.with_mlp(ZH.attn(window=70), ZH.dense()), ZH.with_mlp(ZH.attn(heads=8, kv_heads=2, dim=90, vdim=70, window=200), ZH.moe(experts=9, groups=3)))):
    one_layer(tmp_path / str(i), layer, dtype, n=300, portions=((150, 129, 1),), target=320, rows=320, pages=40, outliers=i == 1)


@pytest.mark.parametrize("dtype", DTYPES)
def test_no_decoder_sizes_are_special(tmp_path, dtype):
  for i, kw in enumerate((dict(vocab=17, width=33, eps=1e-3), dict(vocab=1500, width=130, eps=1e-6), dict(vocab=40, width=1, eps=1e-2))):
    cfg = ZH.model([ZH.with_mlp(ZH.attn(), None)], **kw)
    w = ZH.random_weights(cfg, i)
    eng, _ = VH.engine(VH.write_model(tmp_path / str(i), cfg, w), dtype=dtype)
    t = VH.tokens(cfg, 20, i)
    ZH.check(VH.run_portions(VH.scheduler(eng), "r", t, (20,)), Z.forward(cfg, w, t), dtype)
    eng.close()


def test_other_norm_places(tmp_path, monkeypatch):
  """RMS norms in front only and on both sides, tanh norms behind only: the same kernels under other switches, against the equations written out here."""
  arch = importlib.import_module("maxtext-indextts2_amd.architectures")
  base = ZH.model([ZH.with_mlp(ZH.attn(), ZH.dense()), ZH.with_mlp(ZH.attn(window=20), ZH.moe())])
  t = VH.tokens(base, 30, 3)
  for i, (kind, places) in enumerate(((0, 1), (0, 3), (1, 2), (1, 1))):
    w = ZH.random_weights(base, 20 + i)
    before = lambda n: n if places & 1 else None
    after = lambda n: None if not places & 2 else n + "b" if places == 3 else n
    if places != 3:
      w = {k: v for k, v in w.items() if "norm1b" not in k and "norm2b" not in k}
    if kind == 0:
      w = {k: v for k, v in w.items() if not ("norm" in k and k.endswith((".alpha", ".b")))}
    eps = base["norm"]["eps"]

    def norm(x, n, w=w, kind=kind):
      if n is None:
        return x
      return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps) * (1 + w[n]) if kind == 0 else np.tanh(w[n + ".alpha"] * x) * w[n] + w[n + ".b"]

    x = w["embed"][t]
    for j, l in enumerate(base["layers"]):
      p = f"l{j}."
      x = x + norm(Z.attention(norm(x, before(p + "norm1") and p + "norm1"), Z.under(w, p + "mix."), l["mixer"], eps), after(p + "norm1"))
      x = x + norm(Z.feed_forward(norm(x, before(p + "norm2") and p + "norm2"), Z.under(w, p + "mlp."), l["mlp"]), after(p + "norm2"))
    want = Z.linear(w["head"], norm(x, "final.norm"))
    monkeypatch.setitem(arch.ARCHITECTURES, "VazilornVariant", lambda c, shapes, kind=kind, places=places: dict(
        arch.vazilorn_keys(c, shapes), hybrid_norm_kind=kind, hybrid_norm_places=places))
    eng, _ = VH.engine(VH.write_model(tmp_path / str(i), dict(base, architecture="VazilornVariant"), w))
    ZH.check(VH.run_portions(VH.scheduler(eng), "r", t, (17, 1)), want, "float32", (kind, places))
    eng.close()


# ---------------------------------------------------------------------------------------------------- edges that random weights would hide
def marked_model(window, rng, **kw):
  """One layer in which the key of one marked token stands out for every query, whatever the distance: what turns carries little of it.  -> (cfg,
  weights, the mark)."""
  cfg = ZH.model([ZH.with_mlp(ZH.attn(heads=4, kv_heads=2, dim=16, vdim=16, window=window, dims=4, scale=1.0), None)], **kw)
  w = ZH.random_weights(cfg, 3)
  mark, E = 7, cfg["width"]
  d = rng.standard_normal(E)
  d /= np.linalg.norm(d)
  # behind the tanh norm (slope 1, scale 1, no offset) ordinary tokens have +1 along d's signs in the first half of the features, the mark in the second half
  sign = np.sign(d)
  w["l0.norm1"], w["l0.norm1.b"], w["l0.norm1.alpha"] = np.ones(E), np.zeros(E), np.array(1.0)
  common, special = np.arange(E) < 12, (np.arange(E) >= 12) & (np.arange(E) < 24)
  w["embed"][:, common] = 2.0 * sign[common]
  w["embed"][:, special] = 0.0
  w["embed"][mark, special] = 2.0 * sign[special]
  qdir, E16 = rng.standard_normal(16), 16
  qdir[:4] = 0.0
  qdir /= np.linalg.norm(qdir)
  for t, heads, feats, gain in (("q", 4, common, 3.0), ("k", 2, special, 3.0)):
    m = 0.15 * w[f"l0.mix.{t}"].reshape(heads, E16, E)
    m[:, :, common | special] = 0.0
    m[:, :, feats] += gain * qdir[None, :, None] * sign[None, None, feats]
    w[f"l0.mix.{t}"] = m.reshape(heads * E16, E)
    w[f"l0.mix.{t}.norm"] = np.full(16, 1.3)
  w["l0.mix.sink"] = np.full(4, 2.0)
  return cfg, ZH.rounded(w), mark


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("window", [37, 64, 70])
def test_window_edge_stands_out(tmp_path, dtype, window):
  """Rows at distance window - 1 still see the marked token, rows at distance window do not -- across page borders, in one prompt, in portions and decoded."""
  n = 130
  cfg, w, mark = marked_model(window, np.random.default_rng(4))
  eng, _ = VH.engine(VH.write_model(tmp_path, cfg, w), dtype=dtype, pages=24, target=160, rows=160)
  for place in (0, 7, 8, 23, 40):
    t = VH.tokens(cfg, n, 9)
    t[t == mark] = 8
    t[place] = mark
    u = t.copy()
    u[place] = 8
    want = Z.forward(cfg, w, t)
    seen = VH.rel(Z.forward(cfg, w, u), want)                    # how much the marked token matters at every row
    assert seen[place + window - 1] > 0.05 and seen[place + window] < 1e-9, seen[place + window - 2:place + window + 2]
    for cuts in ((n,), (place + window - 1, 1), (place + window, 1), (40, 2)):
      s = VH.scheduler(eng)
      got = VH.run_portions(s, "r", t, cuts)
      ZH.check(got, want, dtype, (place, cuts))
      edge = slice(place + window - 2, place + window + 2)
      assert (VH.rel(got, want)[edge] < 0.4 * seen[place + window - 1]).all(), (place, cuts, VH.rel(got, want)[edge], seen[edge])
      s.release("r")
  eng.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_far_keys_stand_out(tmp_path, dtype):
  """A marked token hundreds of positions back, next to page borders and tile borders, seen from the end of a long prompt and from decoded tokens (keys
  in several splits)."""
  n = 700
  cfg, w, mark = marked_model(5000, np.random.default_rng(6))
  eng, _ = VH.engine(VH.write_model(tmp_path, cfg, w), dtype=dtype, pages=100, target=720, rows=720)
  for place in (0, 63, 64, 255, 300):
    t = VH.tokens(cfg, n, 9)
    t[t == mark] = 8
    t[place] = mark
    want = Z.forward(cfg, w, t)
    u = t.copy()
    u[place] = 8
    assert VH.rel(Z.forward(cfg, w, u), want)[-20:].min() > 0.02
    for cuts in ((n,), (n - 9, 1), (257, 129, 31, 2)):
      s = VH.scheduler(eng)
      ZH.check(VH.run_portions(s, "r", t, cuts), want, dtype, (place, cuts))
      s.release("r")
  eng.close()


# ---------------------------------------------------------------------------------------------------- cache and batches
@pytest.fixture(scope="module", params=DTYPES)
def whole(request, tmp_path_factory):
  cfg = ZH.mixed_model()
  w = ZH.random_weights(cfg, 5)
  eng, params = VH.engine(VH.write_model(tmp_path_factory.mktemp("vazilorn"), cfg, w), dtype=request.param, slots=3, pages=30)
  yield cfg, w, eng, params, request.param
  eng.close()


def test_prompt_token_by_token_and_portions(whole):
  cfg, w, eng, _, dtype = whole
  t = VH.tokens(cfg, 80, 6)
  want = Z.forward(cfg, w, t)
  s, base = VH.scheduler(eng), None
  for cuts in ((80,), (1,), (2,), (3, 5), (16,), (17, 1, 2, 30), (79, 1)):
    got = VH.run_portions(s, "r", t, cuts)
    ZH.check(got, want, dtype, cuts)
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
    ZH.check(VH.run_portions(s, "r", t, (n,)), Z.forward(cfg, w, t), dtype, n)
    s.release("r")


def test_unequal_requests_in_one_batch(whole):
  """Prompts, portions and single tokens of three requests in every step, one request paused for some steps."""
  cfg, w, eng, _, dtype = whole
  toks = {"a": VH.tokens(cfg, 70, 31), "b": VH.tokens(cfg, 33, 32), "c": VH.tokens(cfg, 52, 33)}
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
    ZH.check(np.concatenate(got[k]), Z.forward(cfg, w, toks[k]), dtype, k)
    s.release(k)


@pytest.mark.parametrize("dtype", DTYPES)
def test_slots_and_pages_are_used_again(tmp_path, dtype):
  """A pool for one and a half requests and two slots: every new request takes pages that another one has left full."""
  cfg = ZH.mixed_model()
  w = ZH.random_weights(cfg, 8)
  eng, _ = VH.engine(VH.write_model(tmp_path, cfg, w), dtype=dtype, slots=2, pages=9, page=8, target=64, rows=64)
  s = VH.scheduler(eng)
  for i, (n, cuts) in enumerate(((48, (48,)), (5, (1,)), (33, (9,)), (64, (30, 1)), (2, (2,)), (40, (39, 1)))):
    t = VH.tokens(cfg, n, 40 + i)
    ZH.check(VH.run_portions(s, i, t, cuts), Z.forward(cfg, w, t), dtype, i)
    s.release(i)
  t = VH.tokens(cfg, 60, 50)
  with pytest.raises(ValueError, match="pool"):
    s.step([("x", t, []), ("y", t, [])])
  eng.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_large_mixed_steps_and_passes(tmp_path, dtype):
  """Steps of some hundred rows made of long portions beside single tokens, also where a step is cut into passes of 128 rows."""
  cfg = ZH.mixed_model()
  w = ZH.random_weights(cfg, 5)
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
      ZH.check(np.concatenate(got[k]), Z.forward(cfg, w, toks[k]), dtype, (rows, k))
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
  cfg = ZH.mixed_model()
  w = ZH.random_weights(cfg, 10)
  eng, params = VH.engine(VH.write_model(tmp_path, cfg, w), slots=1, pages=60, target=420, rows=32)
  t = VH.tokens(cfg, 9, 3)
  out = decode_greedy(eng, params, t, 400)
  assert_greedy(out, Z.forward(cfg, w, np.concatenate([t, out])[:-1])[len(t) - 1:])
  eng.close()


def test_greedy_generation_by_every_entry_point(tmp_path, capsys):
  """MaxEngine.prefill / insert / generate (graph and eager), StepScheduler.generate and the command line give the restatement's greedy tokens."""
  cfg = ZH.mixed_model()
  w = ZH.random_weights(cfg, 11)
  path = VH.write_model(tmp_path, cfg, w)
  prompts = {i: VH.tokens(cfg, (13, 30, 4, 21, 8)[i], 60 + i) for i in range(5)}
  N = 20
  eng, params = VH.engine(path, slots=3)
  eager, eparams = VH.engine(path, slots=3, ixt_use_hip_graph=False)
  by_steps = VH.scheduler(eng).generate({k: v.tolist() for k, v in prompts.items()}, N, portion=6)
  for i, p in prompts.items():
    out = np.array(by_steps[i])
    assert_greedy(out, Z.forward(cfg, w, np.concatenate([p, out])[:-1])[len(p) - 1:])
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
  cfg = ZH.mixed_model()
  path = VH.write_model(tmp_path, cfg, ZH.random_weights(cfg, 12))
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
  cfg = ZH.mixed_model()
  w = ZH.random_weights(cfg, 13)
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
    assert_greedy(outs[i], Z.forward(cfg, w, np.concatenate([toks[i], outs[i]])[:-1])[lens[i] - 1:])
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
  return np.stack(got), np.stack([Z.forward(cfg, w, s[:-1])[-steps:] for s in seqs], axis=1)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(ATTENTIONS))
def test_decode_step_alone(tmp_path, name, dtype):
  """The decode step's own attention (queries, key and value straight from the projection) at every size: positions around page and tile borders."""
  cfg = ZH.model([ZH.with_mlp(ATTENTIONS[name], None)])
  w = ZH.random_weights(cfg, 2)
  eng, params = VH.engine(VH.write_model(tmp_path, cfg, w), dtype=dtype, slots=3, pages=40, target=90, rows=80)
  got, want = decode_all(cfg, w, eng, params, (1, 61, 36), 9, 300)
  for i in range(3):
    ZH.check(got[:, i], want[:, i], dtype, (name, i))
  eng.close()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("slots", [40, 130])
def test_many_slots_decode_together(tmp_path, slots, dtype):
  """Sequences of unequal length: the decode step's forms for some tens and for more than 128 rows."""
  cfg = ZH.mixed_model()
  w = ZH.random_weights(cfg, 5)
  eng, params = VH.engine(VH.write_model(tmp_path, cfg, w), dtype=dtype, slots=slots, pages=5 * slots, target=40, rows=32)
  got, want = decode_all(cfg, w, eng, params, [1 + (7 * i) % 30 for i in range(slots)], 4, 200)
  for k in range(4):
    ZH.check(got[k], want[k], dtype, k)
  eng.close()


def test_chunked_prefill_prompt_logp_and_sampling_ranges(tmp_path):
  cfg = ZH.mixed_model()
  w = ZH.random_weights(cfg, 14)
  eng, params = VH.engine(VH.write_model(tmp_path, cfg, w), slots=2)
  t = VH.tokens(cfg, 50, 90)
  want = Z.forward(cfg, w, t)
  logp = want - np.log(np.exp(want - want.max(axis=1, keepdims=True)).sum(axis=1, keepdims=True)) - want.max(axis=1, keepdims=True)
  prefix, _ = eng.prefill(params=params, padded_tokens=t[:30], true_length=30, slot=1, return_prompt_logp=True)
  assert np.abs(prefix["prompt_logp"].cpu().numpy()[0] - logp[np.arange(30), t[:30]]).max() < 1e-3
  old = H.maxengine_module().ExistingPrefix(cache=prefix["cache"], common_prefix_tokens=t[:30])
  for _ in range(2):                                    # (keys and values can be written again: a portion may be repeated)
    nxt, _ = eng.prefill(params=params, existing_prefix=old, padded_tokens=t[30:], true_length=20, slot=1)
    ZH.check(nxt["logits"].cpu().numpy().reshape(1, -1), want[49:50], "float32")
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
  cfg = ZH.mixed_model()
  w = ZH.random_weights(cfg, 5)
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
  wa, wb = Z.forward(cfg, w, a), Z.forward(cfg, w, b)
  assert not (tmp_path / "o" / "1.f32").exists()
  ZH.check(load(0), wa[[0, 63]], dtype)
  ZH.check(load(2), np.stack([wa[69], wb[11]]), dtype)
  ZH.check(load(3), wb[11:12], dtype)
