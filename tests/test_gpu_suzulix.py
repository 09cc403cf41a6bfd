"""Suzulix on the GPU against the plain float64 restatement (suzulix_ref): every mechanism alone at many sizes, then the cache, the states, the batch and
the engine's entry points.  float32 is held to rounding of f32 sums, bfloat16 to rounding of its operands (suzulix_helpers.TOL)."""
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
import suzulix_helpers as SH
import suzulix_ref as S
import vilepel_helpers as VH

pytestmark = pytest.mark.gpu
DTYPES = ["float32", "bfloat16"]


def one_layer(tmp_path, layer, dtype, n=50, seed=0, portions=(), alter=None, outliers=False, streams=3, loop=None, **kw):
  """The sum of the streams behind one layer for a prompt (and for the same tokens in portions) against the restatement."""
  cfg = SH.model([layer], streams=streams, loop=loop)
  w = SH.random_weights(cfg, seed)
  if alter is not None:
    alter(w)
    w = SH.rounded(w)
  toks = VH.tokens(cfg, n, seed + 1)
  taps = []
  S.forward(cfg, w, toks, taps)
  want = np.concatenate(taps, axis=1)
  eng, _ = VH.engine(VH.write_model(tmp_path, cfg, w), dtype=dtype, **kw)
  for cuts in ((n,),) + tuple(portions):
    s, got, at, i = VH.scheduler(eng), [], 0, 0
    while at < n:
      m = min(cuts[min(i, len(cuts) - 1)], n - at)
      tap = torch.zeros(len(taps) * m * cfg["width"], device="cuda")
      H.lib.check(eng.lib.ixt_set_residual_tap(eng._ctx, ctypes.c_void_p(tap.data_ptr()), tap.numel()))
      s.step([("r", toks[at:at + m], [])])
      got.append(tap.cpu().numpy().reshape(len(taps), m, -1).transpose(1, 0, 2).reshape(m, -1))
      at, i = at + m, i + 1
    s.release("r")
    r = SH.rel(np.concatenate(got), want)
    if dtype == "float32":
      assert r.max() < 1e-5, (cuts, int(r.argmax()), r.max())
    else:                                           # (a close choice of experts may turn over with rounding)
      assert np.quantile(r, 0.9) < 0.015 and (r.max() < 0.03 or outliers), (cuts, int(r.argmax()), np.quantile(r, 0.9), r.max())
  eng.close()


MIXERS = {
    "attention: one head": SH.attn(heads=1, kv_heads=1, dim=8, vdim=8, dims=8),
    "attention: odd sizes": SH.attn(heads=3, kv_heads=3, dim=23, vdim=17, dims=10),
    "attention: nothing turns": SH.attn(heads=2, kv_heads=2, dims=0),
    "attention: one pair turns": SH.attn(heads=4, kv_heads=2, dims=2),
    "attention: many heads on one": SH.attn(heads=20, kv_heads=1, dim=12, vdim=12, dims=12),
    "attention: more heads than a tile": SH.attn(heads=70, kv_heads=2, dim=8, vdim=4, dims=4),
    "attention: 32": SH.attn(heads=6, kv_heads=2, dim=32, vdim=56, dims=16, softcap=30.0),
    "attention: values wider": SH.attn(heads=4, kv_heads=2, dim=30, vdim=110, dims=30),
    "attention: keys wider": SH.attn(heads=4, kv_heads=4, dim=64, vdim=60, dims=64),
    "attention: 64": SH.attn(heads=6, kv_heads=2, dim=60, vdim=128, dims=32, scale=0.125, diff=0.8),
    "attention: 90": SH.attn(heads=4, kv_heads=1, dim=90, vdim=100, dims=90, scale=0.1),
    "attention: 96": SH.attn(heads=2, kv_heads=2, dim=96, vdim=180, dims=64, scale=0.1),
    "attention: 128": SH.attn(heads=4, kv_heads=2, dim=128, vdim=128, dims=64, scale=0.09),
    "attention: 128 and 256": SH.attn(heads=2, kv_heads=1, dim=120, vdim=250, dims=64, scale=0.09),
    "attention: beyond the tiles": SH.attn(heads=2, kv_heads=1, dim=140, vdim=300, dims=64, scale=0.08),
    "attention: hard cap": SH.attn(softcap=0.5, scale=2.0),
    "attention: far cap": SH.attn(softcap=300.0, scale=0.5),
    "attention: no difference": SH.attn(diff=0.0),
    "latent: one head": SH.latent(heads=1, dim=8, rot=2, vdim=8, rank=16, q_rank=1),
    "latent: odd sizes": SH.latent(heads=3, dim=21, rot=10, vdim=19, rank=41, q_rank=35),
    "latent: many heads": SH.latent(heads=20, dim=8, rot=8, vdim=8, rank=64, q_rank=150),
    "latent: more heads than a tile": SH.latent(heads=70, dim=4, rot=4, vdim=4, rank=32, q_rank=24),
    "latent: rank 200": SH.latent(heads=4, dim=40, rot=48, vdim=36, rank=200, q_rank=300),
    "latent: rank 300": SH.latent(heads=16, dim=16, rot=64, vdim=16, rank=300, q_rank=64),
    "retention: one head": SH.retention(heads=1, dim=8, vdim=8, dims=8),
    "retention: odd sizes": SH.retention(heads=5, dim=23, vdim=17, dims=6),
    "retention: nothing turns": SH.retention(heads=2, dims=0),
    "retention: 64": SH.retention(heads=3, dim=64, vdim=62, dims=48),
    "retention: values wider": SH.retention(heads=2, dim=40, vdim=128, dims=40),
    "retention: keys wider": SH.retention(heads=2, dim=130, vdim=20, dims=64),
    "retention: 128 and 200": SH.retention(heads=2, dim=128, vdim=200, dims=128),
    "retention: 260 and 300": SH.retention(heads=1, dim=260, vdim=300, dims=32),
    "retention: fast and not at all": SH.retention(heads=3, decay=[0.05, 0.75, 1.0]),
}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(MIXERS))
def test_mixer_alone(tmp_path, name, dtype):
  one_layer(tmp_path, SH.with_mlp(MIXERS[name], None), dtype, n=75, portions=((1,), (2,), (33, 2), (7, 1, 40), (64, 11)))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("streams", [1, 2, 4, 5, 16])
def test_streams(tmp_path, streams, dtype):
  for i, mlp in enumerate((None, SH.moe())):
    one_layer(tmp_path / str(i), SH.with_mlp(SH.attn(), mlp), dtype, n=30, portions=((1,), (13, 17)), streams=streams, outliers=True)


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_looped_layer_keeps_a_state_per_pass(tmp_path, dtype):
  for i, layer in enumerate((SH.attn(), SH.latent(), SH.retention())):
    one_layer(tmp_path / str(i), SH.with_mlp(layer, None), dtype, n=40, portions=((1,), (9, 31)), loop={"start": 0, "stop": 1, "times": 3})


MLPS = {"routed": SH.moe(), "no shared unit": SH.moe(shared=0), "one of many": SH.moe(ff=16, experts=72, top=1), "all": SH.moe(ff=130, experts=4, top=4), "one expert": SH.moe(experts=1, top=1),
        "shared unit in parts": SH.moe(ff=20, shared=390), "shared unit of one": SH.moe(ff=140, shared=1), "eight and the gate": SH.moe(experts=8, top=2), "sixteen": SH.moe(experts=16, top=5)}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(MLPS))
def test_feed_forwards(tmp_path, name, dtype):
  one_layer(tmp_path, SH.with_mlp(SH.retention(), MLPS[name]), dtype, n=70, portions=((1,), (9, 61)), outliers=True)


def test_router_logits_from_level_to_far_apart(tmp_path):
  for i, f in enumerate((0.0, 30.0)):
    def spread(w, f=f):
      w["l0.mlp.router"] *= f
    one_layer(tmp_path / str(i), SH.with_mlp(SH.attn(), SH.moe(experts=9, top=4)), "float32", n=40, portions=((1,),), alter=spread)


@pytest.mark.parametrize("dtype", DTYPES)
def test_many_rows_take_the_prompt_kernels(tmp_path, dtype):
  """300 rows in one pass: the ring GEMMs, tall attention tiles, several chunks of the recurrence and 128-row expert groups."""
  for i, layer in enumerate((SH.with_mlp(SH.attn(), SH.moe(experts=9)), SH.with_mlp(SH.attn(heads=8, kv_heads=2, dim=60, vdim=120, dims=60, scale=0.1), None), SH.with_mlp(SH.latent(), SH.moe(shared=200)),
                             SH.with_mlp(SH.retention(heads=2, dim=90, vdim=100, decay=[0.97, 1 - 2.0 ** -10]), None), SH.with_mlp(SH.retention(dim=20, vdim=20), SH.moe(shared=0)))):
    one_layer(tmp_path / str(i), layer, dtype, n=300, portions=((150, 129, 1),), target=320, rows=320, pages=40, outliers=layer["mlp"] is not None)


@pytest.mark.parametrize("dtype", DTYPES)
def test_no_decoder_sizes_are_special(tmp_path, dtype):
  for i, kw in enumerate((dict(vocab=17, width=33, eps=1e-3, logit_scale=0.3), dict(vocab=1500, width=130, eps=1e-6, streams=2), dict(vocab=300, width=2050, streams=6, scale=1.0),
                          dict(vocab=300, width=2052, streams=2), dict(vocab=100, width=4100, streams=4))):
    cfg = SH.model([SH.with_mlp(SH.attn(), None), SH.with_mlp(SH.retention(), SH.moe(experts=3, top=3))], **kw)
    w = SH.random_weights(cfg, i)
    eng, _ = VH.engine(VH.write_model(tmp_path / str(i), cfg, w), dtype=dtype)
    t = VH.tokens(cfg, 20, i)
    SH.check(VH.run_portions(VH.scheduler(eng), "r", t, (20,)), S.forward(cfg, w, t), dtype, kw)
    eng.close()


def test_other_norms_and_rotations_of_the_older_mixers(tmp_path, monkeypatch):
  """Layer norms on one residual sum, in front, behind and on both sides; heads with normed queries and keys that turn in halves: the same switches in
  another design, against the equations written out here."""
  import vazilorn_helpers as ZH
  import vazilorn_ref as Z
  arch = importlib.import_module("maxtext-indextts2_amd.architectures")
  dataclasses = importlib.import_module("dataclasses")
  base = ZH.model([ZH.with_mlp(ZH.attn(scaling=None), ZH.dense()), ZH.with_mlp(ZH.attn(window=20, scaling=None), ZH.moe())])
  t, eps = VH.tokens(base, 30, 3), base["norm"]["eps"]
  monkeypatch.setattr(Z, "rotate_first", S.rotate_halves)
  for i, places in enumerate((1, 2, 3)):
    w = {k: v for k, v in ZH.random_weights(base, 20 + i).items() if not ("norm" in k and k.endswith(".alpha")) and (places == 3 or "norm1b" not in k and "norm2b" not in k)}
    before = lambda x, n, w=w, places=places: S.layer_norm(x, w[n], w[n + ".b"], eps) if places & 1 else x
    after = lambda x, n, w=w, places=places: S.layer_norm(x, w[n + ("b" if places == 3 else "")], w[n + ("b" if places == 3 else "") + ".b"], eps) if places & 2 else x
    x = w["embed"][t]
    for j, l in enumerate(base["layers"]):
      p = f"l{j}."
      x = x + after(Z.attention(before(x, p + "norm1"), S.under(w, p + "mix."), l["mixer"], eps), p + "norm1")
      x = x + after(Z.feed_forward(before(x, p + "norm2"), S.under(w, p + "mlp."), l["mlp"]), p + "norm2")
    want = S.linear(w["head"], S.layer_norm(x, w["final.norm"], w["final.norm.b"], eps))

    def reader(c, shapes, places=places):
      keys = arch.vazilorn_keys(c, shapes)
      return dict(keys, hybrid_norm_kind=arch.NORM_LAYER, hybrid_norm_places=places, hybrid_layers=tuple(dataclasses.replace(l, rope_pairs=arch.ROPE_HALVES) for l in keys["hybrid_layers"]))

    monkeypatch.setitem(arch.ARCHITECTURES, "VazilornVariant", reader)
    eng, _ = VH.engine(VH.write_model(tmp_path / str(i), dict(base, architecture="VazilornVariant"), w))
    SH.check(VH.run_portions(VH.scheduler(eng), "r", t, (17, 1)), want, "float32", places)
    eng.close()


# ---------------------------------------------------------------------------------------------------- far tokens that random weights would hide
def marked_model(kind, rng, eps=3e-5):
  """One layer in which the key of one marked token stands out for every query, whatever the distance -> (cfg, weights, the mark)."""
  layer = {"attention": SH.attn(heads=4, kv_heads=2, dim=16, vdim=16, dims=4, scale=1.0, softcap=18.0), "latent": SH.latent(heads=4, dim=16, rot=4, vdim=16, rank=24, q_rank=16, scale=1.0),
           "retention": SH.retention(heads=4, dim=16, vdim=16, dims=4, decay=[1 - 2.0 ** -12, 1 - 2.0 ** -11, 1 - 2.0 ** -10, 1.0])}[kind]
  cfg = SH.model([SH.with_mlp(layer, None)], eps=eps)
  w, mark, E = SH.random_weights(cfg, 3), 7, cfg["width"]
  common, special = np.arange(E) < 12, (np.arange(E) >= 12) & (np.arange(E) < 24)
  sign = np.sign(rng.standard_normal(E))
  sign[common] -= sign[common].mean()
  sign[special] -= sign[special].mean()
  w["embed"][:, common] = 2.0 * sign[common]               # every token has this, only the mark has that
  w["embed"][:, special] = 0.0
  w["embed"][mark, special] = 3.0 * sign[special]
  w["l0.norm1"], w["l0.norm1.b"] = np.ones(E), np.zeros(E)
  q = rng.standard_normal(16)
  q[:4] = 0.0
  q /= np.linalg.norm(q)

  def point(name, rows, direction, feats, gain, noise=0.15):
    """The named matrix: small on the two groups of features, `direction` (of `rows`) for what is in `feats`."""
    m = noise * w[name].reshape(-1, rows, E)
    m[:, :, common | special] = 0.0
    if feats is not None:
      m[:, :, feats] += gain * direction[None, :, None] * sign[None, None, feats] / 12
    w[name] = m.reshape(w[name].shape)

  if kind == "attention":                                  # the first map looks for the mark, the second does not
    both = np.concatenate([q, np.zeros(16)])
    point("l0.mix.q", 32, both, common, 5.0)
    point("l0.mix.k", 32, both, special, 5.0)
  elif kind == "retention":
    point("l0.mix.q", 16, q, common, 5.0)
    point("l0.mix.k", 16, q, special, 60.0)
  else:
    first = lambda n: np.eye(n)[0]
    point("l0.mix.dq", 16, first(16), common, 8.0)
    point("l0.mix.dkv", 28, first(28), special, 30.0, 0.6)
    w["l0.mix.uq"] = 0.15 * w["l0.mix.uq"]
    w["l0.mix.uq"].reshape(4, 20, 16)[:, :16, 0] += 1.5 * q
    w["l0.mix.uk"] = 0.15 * w["l0.mix.uk"]
    w["l0.mix.uk"].reshape(4, 16, 24)[:, :, 0] += 1.2 * q
  return cfg, SH.rounded(w), mark


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind", ["attention", "latent", "retention"])
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
    want = S.forward(cfg, w, t)
    u = t.copy()
    u[place] = 8
    assert SH.rel(S.forward(cfg, w, u), want)[-20:].min() > 3 * SH.TOL["bfloat16"], SH.rel(S.forward(cfg, w, u), want)[-20:]
    for cuts in ((n,), (n - 9, 1), (257, 129, 31, 2)):
      s = VH.scheduler(eng)
      SH.check(VH.run_portions(s, "r", t, cuts), want, dtype, (place, cuts))
      s.release("r")
    st = eng.init_decode_state(materialize_logits=True)    # the decode step's own kernels
    padded = np.zeros(eng.max_prefill_length, np.int32)
    padded[:n] = t
    prefix, first = eng.prefill(params=params, padded_tokens=padded, true_length=n, slot=0)
    st = eng.insert(prefix, st, 0)
    st, _ = eng.generate(params, st)
    seq = np.concatenate([t, [int(first.data[0, 0])]])
    SH.check(np.concatenate([prefix["logits"].cpu().numpy().reshape(1, -1), st["logits"].cpu().numpy().reshape(1, -1)]), S.forward(cfg, w, seq)[-2:], dtype, (place, "step"))
    eng.release_pages(0)
  eng.close()


# ---------------------------------------------------------------------------------------------------- cache and batches
@pytest.fixture(scope="module", params=DTYPES)
def whole(request, tmp_path_factory):
  cfg = SH.mixed_model()
  w = SH.random_weights(cfg, 5)
  eng, params = VH.engine(VH.write_model(tmp_path_factory.mktemp("suzulix"), cfg, w), dtype=request.param, slots=3, pages=30)
  yield cfg, w, eng, params, request.param
  eng.close()


def test_prompt_token_by_token_and_portions(whole):
  cfg, w, eng, _, dtype = whole
  t = VH.tokens(cfg, 80, 6)
  want = S.forward(cfg, w, t)
  s, base = VH.scheduler(eng), None
  for cuts in ((80,), (1,), (2,), (3, 5), (16,), (17, 1, 2, 30), (79, 1)):
    got = VH.run_portions(s, "r", t, cuts)
    SH.check(got, want, dtype, cuts)
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
    SH.check(VH.run_portions(s, "r", t, (n,)), S.forward(cfg, w, t), dtype, n)
    s.release("r")


def test_unequal_requests_in_one_batch(whole):
  """Prompts, portions and single tokens of three requests in every step, one request paused for some steps."""
  cfg, w, eng, _, dtype = whole
  toks = {"a": VH.tokens(cfg, 70, 48), "b": VH.tokens(cfg, 33, 62), "c": VH.tokens(cfg, 52, 48)}      # (no choice of experts is close in these)
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
    SH.check(np.concatenate(got[k]), S.forward(cfg, w, toks[k]), dtype, k)
    s.release(k)


@pytest.mark.parametrize("dtype", DTYPES)
def test_slots_and_pages_are_used_again(tmp_path, dtype):
  """A pool for one and a half requests and two slots: every new request takes pages that another one has left full."""
  cfg = SH.mixed_model()
  w = SH.random_weights(cfg, 8)
  eng, _ = VH.engine(VH.write_model(tmp_path, cfg, w), dtype=dtype, slots=2, pages=9, page=8, target=64, rows=64)
  s = VH.scheduler(eng)
  for i, (n, cuts) in enumerate(((48, (48,)), (5, (1,)), (33, (9,)), (64, (30, 1)), (2, (2,)), (40, (39, 1)))):
    t = VH.tokens(cfg, n, 40 + i)
    SH.check(VH.run_portions(s, i, t, cuts), S.forward(cfg, w, t), dtype, i)
    s.release(i)
  t = VH.tokens(cfg, 60, 50)
  with pytest.raises(ValueError, match="pool"):
    s.step([("x", t, []), ("y", t, [])])
  eng.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_large_mixed_steps_and_passes(tmp_path, dtype):
  """Steps of some hundred rows made of long portions beside single tokens, also where a step is cut into passes of 128 rows."""
  cfg = SH.mixed_model()
  w = SH.random_weights(cfg, 5)
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
      SH.check(np.concatenate(got[k]), S.forward(cfg, w, toks[k]), dtype, (rows, k))
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
  cfg = SH.mixed_model()
  w = SH.random_weights(cfg, 10)
  eng, params = VH.engine(VH.write_model(tmp_path, cfg, w), slots=1, pages=60, target=420, rows=32)
  t = VH.tokens(cfg, 9, 3)
  out = decode_greedy(eng, params, t, 400)
  assert_greedy(out, S.forward(cfg, w, np.concatenate([t, out])[:-1])[len(t) - 1:])
  eng.close()


def test_greedy_generation_by_every_entry_point(tmp_path, capsys):
  """MaxEngine.prefill / insert / generate (graph and eager), StepScheduler.generate and the command line give the restatement's greedy tokens."""
  cfg = SH.mixed_model()
  w = SH.random_weights(cfg, 11)
  path = VH.write_model(tmp_path, cfg, w)
  prompts = {i: VH.tokens(cfg, (13, 30, 4, 21, 8)[i], 60 + i) for i in range(5)}
  N = 20
  eng, params = VH.engine(path, slots=3)
  eager, eparams = VH.engine(path, slots=3, ixt_use_hip_graph=False)
  by_steps = VH.scheduler(eng).generate({k: v.tolist() for k, v in prompts.items()}, N, portion=6)
  for i, p in prompts.items():
    out = np.array(by_steps[i])
    assert_greedy(out, S.forward(cfg, w, np.concatenate([p, out])[:-1])[len(p) - 1:])
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
  cfg = SH.mixed_model()
  path = VH.write_model(tmp_path, cfg, SH.random_weights(cfg, 12))
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
  cfg = SH.mixed_model()
  w = SH.random_weights(cfg, 13)
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
    assert_greedy(outs[i], S.forward(cfg, w, np.concatenate([toks[i], outs[i]])[:-1])[lens[i] - 1:])
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
  return np.stack(got), np.stack([S.forward(cfg, w, s[:-1])[-steps:] for s in seqs], axis=1)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(MIXERS))
def test_decode_step_alone(tmp_path, name, dtype):
  """The decode step's own attention (queries, key and value straight from the projection) at every size: positions around page and tile borders."""
  cfg = SH.model([SH.with_mlp(MIXERS[name], None)])
  w = SH.random_weights(cfg, 2)
  eng, params = VH.engine(VH.write_model(tmp_path, cfg, w), dtype=dtype, slots=3, pages=40, target=90, rows=80)
  got, want = decode_all(cfg, w, eng, params, (1, 61, 36), 9, 300)
  for i in range(3):
    SH.check(got[:, i], want[:, i], dtype, (name, i))
  eng.close()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("slots", [40, 130])
def test_many_slots_decode_together(tmp_path, slots, dtype):
  """Sequences of unequal length: the decode step's forms for some tens and for more than 128 rows."""
  cfg = SH.mixed_model()
  w = SH.random_weights(cfg, 5)
  eng, params = VH.engine(VH.write_model(tmp_path, cfg, w), dtype=dtype, slots=slots, pages=5 * slots, target=40, rows=32)
  got, want = decode_all(cfg, w, eng, params, [1 + (7 * i) % 30 for i in range(slots)], 4, 200)
  for k in range(4):
    SH.check(got[k], want[k], dtype, k)
  eng.close()


def test_chunked_prefill_prompt_logp_and_sampling_ranges(tmp_path):
  cfg = SH.mixed_model()
  w = SH.random_weights(cfg, 14)
  eng, params = VH.engine(VH.write_model(tmp_path, cfg, w), slots=2)
  t = VH.tokens(cfg, 50, 90)
  want = S.forward(cfg, w, t)
  logp = want - np.log(np.exp(want - want.max(axis=1, keepdims=True)).sum(axis=1, keepdims=True)) - want.max(axis=1, keepdims=True)
  prefix, _ = eng.prefill(params=params, padded_tokens=t[:30], true_length=30, slot=1, return_prompt_logp=True)
  assert np.abs(prefix["prompt_logp"].cpu().numpy()[0] - logp[np.arange(30), t[:30]]).max() < 1e-3
  old = H.maxengine_module().ExistingPrefix(cache=prefix["cache"], common_prefix_tokens=t[:30])
  nxt, _ = eng.prefill(params=params, existing_prefix=old, padded_tokens=t[30:], true_length=20, slot=1)
  SH.check(nxt["logits"].cpu().numpy().reshape(1, -1), want[49:50], "float32")
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
  cfg = SH.mixed_model()
  w = SH.random_weights(cfg, 5)
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
  wa, wb = S.forward(cfg, w, a), S.forward(cfg, w, b)
  assert not (tmp_path / "o" / "1.f32").exists()
  SH.check(load(0), wa[[0, 63]], dtype)
  SH.check(load(2), np.stack([wa[69], wb[11]]), dtype)
  SH.check(load(3), wb[11:12], dtype)
