"""Vilepel on the GPU against the plain float64 restatement (vilepel_ref): every mechanism alone at many sizes, then the cache, the states, the batch
and the engine's entry points.  float32 is held to rounding of f32 sums, bfloat16 to rounding of its operands (vilepel_helpers.TOL)."""
import ctypes
import importlib

import numpy as np
import pytest
import torch

import helpers as H
import vilepel_helpers as VH
import vilepel_ref as V

pytestmark = pytest.mark.gpu
DTYPES = ["float32", "bfloat16"]


def bf16_values(w):
  return {k: torch.from_numpy(v).to(torch.bfloat16).to(torch.float64).numpy() for k, v in w.items()}


def one_layer(tmp_path, layer, dtype, n=50, seed=0, portions=(), alter=None, **kw):
  """Residual stream behind one layer for a prompt (and for the same tokens in portions) against the restatement."""
  cfg = VH.model([layer])
  w = VH.random_weights(cfg, seed)
  if alter is not None:
    alter(w)
    w = bf16_values(w)
  toks = VH.tokens(cfg, n, seed + 1)
  want = []
  V.forward(cfg, w, toks, want)
  want = want[0]
  eng, _ = VH.engine(VH.write_model(tmp_path, cfg, w), dtype=dtype, **kw)
  for cuts in ((n,),) + tuple(portions):
    s, got, at, i = VH.scheduler(eng), [], 0, 0
    while at < n:
      m = min(cuts[min(i, len(cuts) - 1)], n - at)
      tap = torch.zeros(m * cfg["width"], device="cuda")
      VH.H.lib.check(eng.lib.ixt_set_residual_tap(eng._ctx, ctypes.c_void_p(tap.data_ptr()), tap.numel()))
      s.step([("r", toks[at:at + m], [])])
      got.append(tap.cpu().numpy().reshape(m, -1))
      at, i = at + m, i + 1
    s.release("r")
    r = VH.rel(np.concatenate(got), want)
    if dtype == "float32":
      assert r.max() < 1e-5, (cuts, int(r.argmax()), r.max())
    else:
      assert np.quantile(r, 0.9) < 0.02 and (r.max() < 0.06 or layer["mlp"] and layer["mlp"]["kind"] == "moe"), (cuts, int(r.argmax()), r.max())
  eng.close()


LATENTS = {
    "one head": VH.latent(heads=1, dim=8, rot=2, vdim=8, rank=16, window=4),
    "odd sizes": VH.latent(heads=3, dim=24, rot=16, vdim=20, rank=40, window=11),
    "window 1": VH.latent(heads=2, dim=10, rot=4, vdim=6, rank=24, window=1),
    "window past the end": VH.latent(heads=6, dim=16, rot=32, vdim=16, rank=96, window=1000),
    "many heads": VH.latent(heads=20, dim=8, rot=8, vdim=8, rank=64, window=33),
    "more heads than a tile": VH.latent(heads=70, dim=4, rot=4, vdim=4, rank=32, window=17),
    "rank 200, rot 48": VH.latent(heads=4, dim=40, rot=48, vdim=36, rank=200, window=31),
    "rank 300": VH.latent(heads=16, dim=16, rot=64, vdim=16, rank=300, window=40),
    "rank 520": VH.latent(heads=2, dim=16, rot=16, vdim=16, rank=520, window=30),
    "rot 96": VH.latent(heads=2, dim=16, rot=96, vdim=16, rank=48, window=30),
}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(LATENTS))
def test_latent_attention_alone(tmp_path, name, dtype):
  one_layer(tmp_path, VH.with_mlp(LATENTS[name], None), dtype, n=75, portions=((1,), (33, 2), (7, 1, 40)))


DELTAS = {
    "one head": VH.delta(heads=1, kv_heads=1, dim=8, vdim=8, conv=2),
    "shared keys": VH.delta(heads=6, kv_heads=2, dim=20, vdim=12, conv=4),
    "no taps": VH.delta(heads=2, kv_heads=1, dim=33, vdim=17, conv=1),
    "long taps": VH.delta(heads=2, kv_heads=2, dim=64, vdim=5, conv=7),
    "wide values": VH.delta(heads=2, kv_heads=2, dim=16, vdim=100, conv=3),
    "dim 130": VH.delta(heads=1, kv_heads=1, dim=130, vdim=24, conv=4),
    "dim 260": VH.delta(heads=1, kv_heads=1, dim=260, vdim=16, conv=4),
}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(DELTAS))
def test_gated_delta_rule_alone(tmp_path, name, dtype):
  one_layer(tmp_path, VH.with_mlp(DELTAS[name], None), dtype, n=70, portions=((1,), (2,), (17, 3, 1, 20)))


@pytest.mark.parametrize("dtype", DTYPES)
def test_slow_decay_keeps_early_tokens(tmp_path, dtype):
  """Decays next to 1: the state must carry the first tokens to the end, however the prompt is cut."""
  def slow(w):
    w["l0.mix.dt_bias"] -= 7.0
  one_layer(tmp_path, VH.with_mlp(VH.delta(), None), dtype, n=90, portions=((1,), (16,), (31, 2)), alter=slow)


MLPS = {"dense": VH.dense(), "dense, wide": VH.dense(ff=300, limit=0.7), "moe": VH.moe(), "moe, one of many": VH.moe(ff=16, experts=70, top=1),
        "moe, all": VH.moe(ff=130, experts=3, top=3), "moe, one expert": VH.moe(ff=33, experts=1, top=1)}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(MLPS))
def test_feed_forwards(tmp_path, name, dtype):
  one_layer(tmp_path, VH.with_mlp(VH.latent(), MLPS[name]), dtype, n=70, portions=((1,), (9, 61)))


@pytest.mark.parametrize("dtype", DTYPES)
def test_many_rows_take_the_prompt_kernels(tmp_path, dtype):
  """300 rows in one pass: the ring GEMMs, the tall attention tile and the 128-row expert groups."""
  for i, layer in enumerate((VH.with_mlp(VH.latent(window=70), VH.dense()), VH.with_mlp(VH.delta(), VH.moe(experts=9, top=2)))):
    one_layer(tmp_path / str(i), layer, dtype, n=300, portions=((150, 129, 1),), target=320, rows=320, pages=40)


@pytest.mark.parametrize("dtype", DTYPES)
def test_no_decoder_sizes_are_special(tmp_path, dtype):
  """Vocabulary, width and eps that divide nothing; a model of one layer without feed-forward."""
  for i, kw in enumerate((dict(vocab=17, width=33, eps=1e-3, scale=1.0), dict(vocab=1500, width=130, eps=1e-6, scale=11.0))):
    cfg = VH.model([VH.with_mlp(VH.latent(), None)], **kw)
    w = VH.random_weights(cfg, i)
    eng, _ = VH.engine(VH.write_model(tmp_path / str(i), cfg, w), dtype=dtype)
    t = VH.tokens(cfg, 20, i)
    VH.check(VH.run_portions(VH.scheduler(eng), "r", t, (20,)), V.forward(cfg, w, t), dtype)
    eng.close()


# ---------------------------------------------------------------------------------------------------- edges that random weights would hide
@pytest.mark.parametrize("dtype", DTYPES)
def test_window_edge_and_far_keys_stand_out(tmp_path, dtype):
  """One marked token whose key every query matches: rows at distance window - 1 still see it, rows at distance window do not -- across page
  borders, in one prompt, in portions and decoded."""
  window, n = 37, 90
  cfg = VH.model([VH.with_mlp(VH.latent(heads=2, dim=16, rot=4, vdim=16, rank=32, window=window, scale=1.0), None)], scale=1.0)
  w = VH.random_weights(cfg, 3)
  rng = np.random.default_rng(4)
  mark = 7
  # the marked token's latent points along one direction that all queries share; ordinary tokens have little of it
  d = rng.standard_normal(cfg["width"])
  d /= np.linalg.norm(d)
  emb = w["embed"] - np.outer(w["embed"] @ d, d) + 0.5 * d
  emb[mark] = 25.0 * d + emb[mark]
  w["embed"] = emb
  c = rng.standard_normal(32) / np.sqrt(32)
  w["l0.mix.dkv"][:32] += np.outer(c, d) * 3
  w["l0.mix.dkv"][32:] -= np.outer(w["l0.mix.dkv"][32:] @ d, d)          # (the rotated key part is not normed: the mark stays out of it)
  wq = w["l0.mix.q"].reshape(2, 20, -1)
  wq[:, :16] = 0.05 * wq[:, :16] + np.einsum("hi,e->hie", w["l0.mix.uk"].reshape(2, 16, 32) @ c, d) * 12
  wq[:, 16:] *= 0.1
  w["l0.mix.q"] = wq.reshape(40, -1)
  w = bf16_values(w)
  eng, _ = VH.engine(VH.write_model(tmp_path, cfg, w), dtype=dtype)
  for place in (0, 7, 8, 23, 40):
    t = VH.tokens(cfg, n, 9)
    t[t == mark] = 8
    t[place] = mark
    want, other = V.forward(cfg, w, t), None
    u = t.copy()
    u[place] = 8
    other = V.forward(cfg, w, u)
    seen = VH.rel(other, want)                    # how much the marked token matters at every row
    assert seen[place + window - 1] > 0.05 and seen[place + window] < 1e-9, seen[place + window - 2:place + window + 2]
    for cuts in ((n,), (place + window - 1, 1), (place + window, 1), (40, 2)):
      s = VH.scheduler(eng)
      got = VH.run_portions(s, "r", t, cuts)
      VH.check(got, want, dtype, (place, cuts))
      edge = slice(place + window - 2, place + window + 2)
      assert (VH.rel(got, want)[edge] < 0.4 * seen[place + window - 1]).all(), (place, cuts, VH.rel(got, want)[edge], seen[edge])
      s.release("r")
  eng.close()


# ---------------------------------------------------------------------------------------------------- cache, states, batches
@pytest.fixture(scope="module", params=DTYPES)
def whole(request, tmp_path_factory):
  cfg = VH.mixed_model()
  w = VH.random_weights(cfg, 5)
  path = VH.write_model(tmp_path_factory.mktemp("vilepel"), cfg, w)
  eng, params = VH.engine(path, dtype=request.param, slots=3, pages=30)
  yield cfg, w, path, eng, params, request.param
  eng.close()


def test_prompt_token_by_token_and_portions(whole):
  cfg, w, _, eng, _, dtype = whole
  t = VH.tokens(cfg, 80, 6)
  want = V.forward(cfg, w, t)
  s = VH.scheduler(eng)
  base = None
  for cuts in ((80,), (1,), (2,), (3, 5), (16,), (17, 1, 2, 30), (79, 1)):
    got = VH.run_portions(s, "r", t, cuts)
    VH.check(got, want, dtype, cuts)
    if base is None:
      base = got
    elif dtype == "float32":                     # and among themselves, beyond the restatement
      assert VH.rel(got, base).max() < 3e-5, cuts
    s.release("r")


def test_first_tokens(whole):
  cfg, w, _, eng, _, dtype = whole
  s = VH.scheduler(eng)
  for n in (1, 2, 3, 4):
    t = VH.tokens(cfg, n, 20 + n)
    VH.check(VH.run_portions(s, "r", t, (n,)), V.forward(cfg, w, t), dtype, n)
    s.release("r")


def test_unequal_requests_in_one_batch(whole):
  """Prompts, portions and single tokens of three requests in every step, one request paused for some steps."""
  cfg, w, _, eng, _, dtype = whole
  toks = {"a": VH.tokens(cfg, 70, 31), "b": VH.tokens(cfg, 33, 32), "c": VH.tokens(cfg, 52, 33)}
  plan = [("a", 20), ("b", 1), ("a", 1), ("c", 31), ("b", 2), ("a", 2), ("b", 17), ("c", 1)]
  s, at, got = VH.scheduler(eng), dict.fromkeys(toks, 0), {k: [] for k in toks}
  step = 0
  while any(at[k] < len(toks[k]) for k in toks):
    entries = []
    for i, k in enumerate(toks):
      if (step + i) % 4 == 3 or at[k] == len(toks[k]):
        continue
      n = min(plan[(step * 3 + i) % len(plan)][1], len(toks[k]) - at[k])
      entries.append((k, toks[k][at[k]:at[k] + n], list(range(n))))
      at[k] += n
    step += 1
    if not entries:
      continue
    lg, _ = s.step(entries)
    lg = lg.cpu().numpy()
    for k, x, _ in entries:
      got[k].append(lg[:len(x)])
      lg = lg[len(x):]
  for k in toks:
    VH.check(np.concatenate(got[k]), V.forward(cfg, w, toks[k]), dtype, k)
    s.release(k)


def test_slots_and_pages_are_used_again(tmp_path):
  """A pool for one and a half requests and two slots: every new request takes pages and a state slot that another one has left full."""
  cfg = VH.mixed_model()
  w = VH.random_weights(cfg, 8)
  eng, _ = VH.engine(VH.write_model(tmp_path, cfg, w), slots=2, pages=9, page=8, target=64, rows=64)
  s = VH.scheduler(eng)
  for i in range(6):
    n = (48, 5, 33, 64, 2, 40)[i]
    t = VH.tokens(cfg, n, 40 + i)
    VH.check(VH.run_portions(s, i, t, ((n,), (1,), (9,), (30, 1), (2,), (39, 1))[i]), V.forward(cfg, w, t), "float32", i)
    s.release(i)
  t = VH.tokens(cfg, 60, 50)
  with pytest.raises(ValueError, match="pool"):
    s.step([("x", t, []), ("y", t, [])])
  eng.close()


def test_steps_longer_than_a_pass_are_cut(tmp_path):
  cfg = VH.mixed_model()
  w = VH.random_weights(cfg, 9)
  eng, _ = VH.engine(VH.write_model(tmp_path, cfg, w), rows=16)
  s = VH.scheduler(eng)
  a, b = VH.tokens(cfg, 41, 1), VH.tokens(cfg, 22, 2)
  lg, tok = s.step([("a", a, [40, 3, 17]), ("b", b, [21])])          # places in the caller's order
  wa, wb = V.forward(cfg, w, a), V.forward(cfg, w, b)
  want = np.stack([wa[40], wa[3], wa[17], wb[21]])
  VH.check(lg.cpu().numpy(), want, "float32")
  assert tok.cpu().tolist() == want.argmax(axis=1).tolist()
  eng.close()


def test_long_decoding(tmp_path):
  """400 decoded tokens through ixt_generate: far beyond every window, pages taken one by one."""
  cfg = VH.mixed_model()
  w = VH.random_weights(cfg, 10)
  eng, params = VH.engine(VH.write_model(tmp_path, cfg, w), slots=1, pages=60, target=420, rows=32)
  t = VH.tokens(cfg, 9, 3)
  out = decode_greedy(eng, params, t, 400)
  full = np.concatenate([t, out])
  want = V.forward(cfg, w, full[:-1])[len(t) - 1:]
  assert_greedy(out, want)
  eng.close()


def assert_greedy(out, logits, margin=1e-3):
  """The tokens are the argmax of the restatement's logits wherever its lead is not within rounding."""
  top = np.sort(logits, axis=1)
  clear = top[:, -1] - top[:, -2] > margin
  assert clear.mean() > 0.9 and (np.asarray(out)[clear] == logits.argmax(axis=1)[clear]).all()


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


# ---------------------------------------------------------------------------------------------------- the framework's own entry points
def test_greedy_generation_by_every_entry_point(tmp_path, capsys):
  """MaxEngine.prefill / insert / generate (graph and eager), StepScheduler.generate and the command line give the restatement's greedy tokens."""
  cfg = VH.mixed_model()
  w = VH.random_weights(cfg, 11)
  path = VH.write_model(tmp_path, cfg, w)
  prompts = {i: VH.tokens(cfg, (13, 30, 4, 21, 8)[i], 60 + i) for i in range(5)}
  N = 20
  eng, params = VH.engine(path, slots=3)
  eager, eparams = VH.engine(path, slots=3, ixt_use_hip_graph=False)
  by_steps = VH.scheduler(eng).generate({k: v.tolist() for k, v in prompts.items()}, N, portion=6)
  for i, p in prompts.items():
    out = np.array(by_steps[i])
    want = V.forward(cfg, w, np.concatenate([p, out])[:-1])[len(p) - 1:]
    assert_greedy(out, want)
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
  cfg = VH.mixed_model()
  path = VH.write_model(tmp_path, cfg, VH.random_weights(cfg, 12))
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


def test_packed_prefill_and_inserts_carry_the_state(tmp_path):
  """prefill_concat + insert_partial (page lists and states move), insert into another slot and bulk_insert (both are copied)."""
  cfg = VH.mixed_model()
  w = VH.random_weights(cfg, 13)
  eng, params = VH.engine(VH.write_model(tmp_path, cfg, w), slots=4, pages=40, ixt_staging_groups=3, ixt_max_packed_rows=96)
  lens = [21, 6, 30]
  toks = [VH.tokens(cfg, n, 80 + n) for n in lens]
  flat, start = np.concatenate(toks), np.cumsum([0] + lens[:-1])
  cache, res, _ = eng.prefill_concat(params=params, padded_tokens=flat, decoder_positions=np.concatenate([np.arange(n) for n in lens]), decoder_segment_ids=None,
                                     start_pos=start, true_lengths=lens, num_prompts=3)
  st = eng.insert_partial(res, eng.init_decode_state(), cache, [2, 0, 3], num_prompts=3)
  outs = {i: [int(res["tokens"][i].reshape(-1)[0])] for i in range(3)}
  for _ in range(12):
    st, r = eng.generate(params, st)
    for i, slot in enumerate((2, 0, 3)):
      outs[i].append(int(r.data[slot, 0]))
  for i in range(3):
    assert_greedy(outs[i], V.forward(cfg, w, np.concatenate([toks[i], outs[i]])[:-1])[lens[i] - 1:])
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


def test_chunked_prefill_prompt_logp_and_state_misuse(tmp_path):
  cfg = VH.mixed_model()
  w = VH.random_weights(cfg, 14)
  eng, params = VH.engine(VH.write_model(tmp_path, cfg, w), slots=2)
  t = VH.tokens(cfg, 50, 90)
  want = V.forward(cfg, w, t)
  logp = want - np.log(np.exp(want - want.max(axis=1, keepdims=True)).sum(axis=1, keepdims=True)) - want.max(axis=1, keepdims=True)
  maxengine = H.maxengine_module()
  prefix, _ = eng.prefill(params=params, padded_tokens=t[:30], true_length=30, slot=1, return_prompt_logp=True)
  assert np.abs(prefix["prompt_logp"].cpu().numpy()[0] - logp[np.arange(30), t[:30]]).max() < 1e-3
  old = maxengine.ExistingPrefix(cache=prefix["cache"], common_prefix_tokens=t[:30])
  nxt, _ = eng.prefill(params=params, existing_prefix=old, padded_tokens=t[30:], true_length=20, slot=1)
  VH.check(nxt["logits"].cpu().numpy().reshape(1, -1), want[49:50], "float32")
  with pytest.raises(ValueError, match="state"):        # the state stands at 50 tokens; it cannot go back to 30
    eng.prefill(params=params, existing_prefix=old, padded_tokens=t[30:], true_length=20, slot=1)
  prefix, _ = eng.prefill(params=params, padded_tokens=t[:30], true_length=30, slot=1)          # from the start it can
  VH.check(prefix["logits"].cpu().numpy().reshape(1, -1), want[29:30], "float32")
  eng.close()


def test_sampling_ranges_and_other_engines_step(tmp_path):
  """The column restriction of the sampler holds here too; and MaxEngine.step serves the llama2 block as well."""
  cfg = VH.mixed_model()
  w = VH.random_weights(cfg, 15)
  eng, _ = VH.engine(VH.write_model(tmp_path, cfg, w))
  t = VH.tokens(cfg, 20, 95)
  want = V.forward(cfg, w, t)[-1]
  eng.set_sampling_ranges([(3, 40), (100, 150)])
  _, tok = VH.scheduler(eng).step([("r", t, [19])])
  allowed = np.full_like(want, -np.inf)
  for a, b in ((3, 40), (100, 150)):
    allowed[a:b] = want[a:b]
  assert tok.cpu().tolist() == [int(allowed.argmax())]
  eng.close()
  c = H.make_config(per_device_batch_size=2.0)
  other, params = H.make_engine(c, H.synth.synth_weights(c, 0))
  toks, n = H.synth.synth_prompt(c.vocab_size, c.max_prefill_predict_length, 1234)
  pre, _ = other.prefill(params=params, padded_tokens=toks, true_length=n, slot=0)
  s = VH.scheduler(other)
  ids = [int(x) for x in np.asarray(toks)[:n]]
  s.step([("a", ids[:5], []), ("b", ids[:9], [])])
  lg, _ = s.step([("b", ids[9:], [n - 10]), ("a", ids[5:6], [])])
  assert torch.equal(lg[0], pre["logits"].reshape(-1))
  other.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_trace_runner(tmp_path, dtype):
  """The trace program, in this process: steps in, one logits file per step out."""
  import contextlib, io, json, sys
  cfg = VH.mixed_model()
  w = VH.random_weights(cfg, 16)
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
  wa, wb = V.forward(cfg, w, a), V.forward(cfg, w, b)
  assert not (tmp_path / "o" / "1.f32").exists()
  VH.check(load(0), wa[[0, 63]], dtype)
  VH.check(load(2), np.stack([wa[69], wb[11]]), dtype)
  VH.check(load(3), wb[11:12], dtype)


@pytest.mark.parametrize("dtype", DTYPES)
def test_large_mixed_steps(tmp_path, dtype):
  """Steps of some hundred rows made of long portions beside single tokens: the prompt kernels with several requests per tile and per launch."""
  cfg = VH.mixed_model()
  w = VH.random_weights(cfg, 18)      # (no routing decision that bf16 inputs alone turn over in the first tokens)
  eng, _ = VH.engine(VH.write_model(tmp_path, cfg, w), dtype=dtype, slots=4, pages=110, target=256, rows=512)
  toks = {k: VH.tokens(cfg, n, 100 + n) for k, n in (("a", 250), ("b", 131), ("c", 9), ("d", 200))}
  s, at, got = VH.scheduler(eng), dict.fromkeys(toks, 0), {k: [] for k in toks}
  for sizes in ((("a", 1), ("c", 5), ("b", 130)), (("a", 150), ("b", 1), ("d", 129), ("c", 1)), (("d", 70), ("c", 3), ("a", 98)), (("a", 1), ("d", 1))):
    lg, _ = s.step([(k, toks[k][at[k]:at[k] + n], list(range(n))) for k, n in sizes])
    lg = lg.cpu().numpy()
    for k, n in sizes:
      got[k].append(lg[:n])
      lg, at[k] = lg[n:], at[k] + n
  for k in toks:
    assert at[k] == len(toks[k])
    VH.check(np.concatenate(got[k]), V.forward(cfg, w, toks[k]), dtype, k)
  eng.close()
