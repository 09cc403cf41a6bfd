"""`bench.py --hybrid SIZES`: prefill and decode rates of hybrid decoders (Vilepel: half latent attention, half gated delta rule; Vazilorn: windowed
attention with sinks and tanh norms; Suzulix: differential attention, retention and latent attention among four streams; Lulenex: chunked attention beside lightning attention, and selective scans) at layer sizes of real models, beside the closest model of the framework at the same width, head count,
feed-forward and number of layers (the llama2 block, or Mixtral for the routed sizes; a unit without a gate gets half as many features more).  Random weights drawn on the device, one GPU, both models in
turn in one process.

Per model: `prefill_packed` = 8 prompts of 256 tokens in one pass (2048 rows), `prefill_long` = one 4096-token prompt in 1024-row chunks,
`decode_<slots>` = generate steps of that many slots at a context of about 1000 tokens.  Every figure is the best of three timed repetitions, each
closed by a device synchronisation.  Prints one JSON line."""
from __future__ import annotations

import json
import os
import tempfile
import time

import numpy as np

PROMPT, PACK, LONG, CHUNK, CONTEXT = 256, 8, 4096, 1024, 1000


def _latent(heads, rank, window, dim=128, rot=64, vdim=128):
  return {"type": "latent_attention", "mixer": {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "kv_rank": rank, "scale": (dim + rot) ** -0.5,
                                                "mask": {"size": window}, "rot": {"base": 10000.0, "dims": rot}}}


def _delta(heads, kv_heads, dim=128, vdim=128):
  return {"type": "channel_delta", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": 4}}


def _dense(ff):
  return {"kind": "dense", "ff": ff, "limit": 7.0}


def _moe(ff, experts, top):
  return {"kind": "moe", "expert": {"ff": ff, "limit": 7.0}, "router": {"experts": experts, "top": top}}


def _model(width, pairs, latent, delta, mlp):
  return {"architecture": "Vilepel", "embedding": {"scale": 1.0}, "norm": {"eps": 1e-5}, "vocab": 32000, "width": width,
          "layers": [dict(l, mlp=mlp) for _ in range(pairs) for l in (delta, latent)]}


def _heads(heads, kv_heads, window, dim=128):
  return {"type": "attention", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": dim ** -0.5, "mask": {"size": window},
                                         "rot": {"base": 500000.0, "dims": dim, "scaling": {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 8192}}}}


def _vazilorn(width, layers, heads, mlp):
  return {"architecture": "Vazilorn", "norm": {"eps": 1e-5}, "vocab": 32000, "width": width, "layers": [dict(heads, mlp=mlp) for _ in range(layers)]}


def _grouped_moe(ff, experts, top, groups, keep, shared):
  return {"kind": "moe", "expert": {"ff": ff}, "shared": {"ff": shared}, "router": {"experts": experts, "top": top, "groups": {"count": groups, "keep": keep}, "scale": 2.5}}


def _suzulix(width, mixers, heads, mlp):
  """Layers of differential attention, retention and latent attention in turn, four streams."""
  dim = 128
  kinds = {"attention": {"heads": heads, "kv_heads": heads // 2, "dim": dim // 2, "vdim": dim, "scale": (dim // 2) ** -0.5, "softcap": 30.0, "diff": 0.5, "rot": {"base": 500000.0, "dims": dim // 2}},
           "retention": {"heads": heads, "dim": dim, "vdim": dim, "decay": [1.0 - 2.0 ** -(5 + 6.0 * i / heads) for i in range(heads)], "rot": {"base": 10000.0, "dims": dim}},
           "latent_attention": {"heads": heads, "dim": dim, "rot_dim": 64, "vdim": dim, "kv_rank": 512, "q_rank": width // 2, "scale": (dim + 64) ** -0.5, "rot": {"base": 10000.0, "dims": 64}}}
  return {"architecture": "Suzulix", "embedding": {"scale": 1.0}, "norm": {"eps": 1e-5}, "vocab": 32000, "width": width, "streams": 4, "logit_scale": 1.0,
          "layers": [{"type": t, "mixer": kinds[t], "mlp": mlp} for t in mixers]}


def _square_moe(ff, experts, top, shared):
  return {"kind": "moe", "expert": {"ff": ff}, "shared": {"ff": shared}, "router": {"experts": experts, "top": top}}


def _lulenex(width, heads, ff, chunk, layers):
  """Attention beside lightning attention and selective scans in turn (the sizes of Mamba's own: inner 2 width, 16 states, rank width / 16)."""
  dim = 128
  both = {"type": "parallel", "mixer": {"left_scale": 1.0, "right_scale": 1.0,
                                        "left": {"heads": heads, "kv_heads": heads // 4, "dim": dim, "vdim": dim, "scale": dim ** -0.5, "mask": {"size": chunk}, "rot": {"base": 500000.0, "dims": dim // 2}},
                                        "right": {"heads": heads, "dim": dim, "vdim": dim, "decay": [1.0 - 2.0 ** -(3 + 6.0 * i / heads) for i in range(heads)]}}}
  scan = {"type": "mamba1", "mixer": {"inner": 2 * width, "state": 16, "dt_rank": width // 16, "conv": 4}}
  return {"architecture": "Lulenex", "norm": {"eps": 1e-5}, "vocab": 32000, "width": width, "loop": None,
          "layers": [dict((both, scan)[i % 2], mlp={"kind": "dense", "ff": ff}) for i in range(layers)]}


# name -> (config.json, keys of the closest model)
SIZES = {
    "w1024": (_model(1024, 4, _latent(8, 256, 512, dim=64), _delta(8, 8), _dense(3584)),
              dict(base_emb_dim=1024, base_num_query_heads=8, base_num_kv_heads=8, base_mlp_dim=3584, base_num_decoder_layers=8)),
    "w2048": (_model(2048, 4, _latent(16, 512, 1024), _delta(16, 16), _dense(7168)),
              dict(base_emb_dim=2048, base_num_query_heads=16, base_num_kv_heads=16, base_mlp_dim=7168, base_num_decoder_layers=8)),
    "w4096-moe": (_model(4096, 1, _latent(32, 512, 1024), _delta(32, 32), _moe(14336, 8, 2)),
                  dict(base_emb_dim=4096, base_num_query_heads=32, base_num_kv_heads=8, base_mlp_dim=14336, base_num_decoder_layers=2, num_experts=8, num_experts_per_tok=2,
                       decoder_block="mixtral")),
    "vazilorn-w1024": (_vazilorn(1024, 8, _heads(8, 8, 512), {"kind": "dense", "ff": 3584}),
                       dict(base_emb_dim=1024, base_num_query_heads=8, base_num_kv_heads=8, base_mlp_dim=3584, base_num_decoder_layers=8)),
    "vazilorn-w2048": (_vazilorn(2048, 8, _heads(16, 16, 1024), {"kind": "dense", "ff": 7168}),
                       dict(base_emb_dim=2048, base_num_query_heads=16, base_num_kv_heads=16, base_mlp_dim=7168, base_num_decoder_layers=8)),
    "vazilorn-w4096-moe": (_vazilorn(4096, 2, _heads(32, 8, 1024), _grouped_moe(14336, 8, 2, 4, 2, 2048)),
                           dict(base_emb_dim=4096, base_num_query_heads=32, base_num_kv_heads=8, base_mlp_dim=14336, base_num_decoder_layers=2, num_experts=8, num_experts_per_tok=2,
                                decoder_block="mixtral")),
    "suzulix-w1024": (_suzulix(1024, ("attention", "retention", "latent_attention") * 2, 8, _square_moe(3584, 8, 2, 3584)),
                      dict(base_emb_dim=1024, base_num_query_heads=8, base_num_kv_heads=4, base_mlp_dim=3584, base_num_decoder_layers=6, num_experts=8, num_experts_per_tok=2,
                           decoder_block="mixtral")),
    "suzulix-w2048": (_suzulix(2048, ("attention", "retention", "latent_attention"), 16, _square_moe(7168, 8, 2, 7168)),
                      dict(base_emb_dim=2048, base_num_query_heads=16, base_num_kv_heads=8, base_mlp_dim=7168, base_num_decoder_layers=3, num_experts=8, num_experts_per_tok=2,
                           decoder_block="mixtral")),
    "suzulix-w4096": (_suzulix(4096, ("attention", "retention", "latent_attention"), 32, _square_moe(14336, 8, 2, 2048)),
                      dict(base_emb_dim=4096, base_num_query_heads=32, base_num_kv_heads=8, base_mlp_dim=14336, base_num_decoder_layers=3, num_experts=8, num_experts_per_tok=2,
                           decoder_block="mixtral")),
    "lulenex-w1024": (_lulenex(1024, 8, 5376, 2048, 8), dict(base_emb_dim=1024, base_num_query_heads=8, base_num_kv_heads=8, base_mlp_dim=3584, base_num_decoder_layers=8)),
    "lulenex-w2048": (_lulenex(2048, 16, 10752, 2048, 8), dict(base_emb_dim=2048, base_num_query_heads=16, base_num_kv_heads=16, base_mlp_dim=7168, base_num_decoder_layers=8)),
    "lulenex-w4096": (_lulenex(4096, 32, 21504, 2048, 2), dict(base_emb_dim=4096, base_num_query_heads=32, base_num_kv_heads=8, base_mlp_dim=14336, base_num_decoder_layers=2)),
}


def _best(fn, n=3):
  import torch  # pylint: disable=import-outside-toplevel
  best = float("inf")
  for _ in range(n):
    torch.cuda.synchronize()
    t = time.perf_counter()
    fn()
    torch.cuda.synchronize()
    best = min(best, time.perf_counter() - t)
  return best


def _measure(make_config, slots_list, opts, log):
  import torch  # pylint: disable=import-outside-toplevel
  from . import _lib, maxengine, synth  # pylint: disable=import-outside-toplevel
  out = {}
  for slots in slots_list:
    last = slots == slots_list[-1]
    cfg = make_config(slots)
    eng = maxengine.MaxEngine(cfg)
    for kv in opts:
      k, v = kv.split("=")
      _lib.check(eng.lib.ixt_set_option(eng._ctx, k.encode(), int(v)))  # pylint: disable=protected-access
    params = eng.load_params(params=synth.DeviceTree(synth.device_tree_spec(cfg)))
    rng = np.random.default_rng(1)
    draw = lambda n: torch.from_numpy(rng.integers(1, cfg.vocab_size, n).astype(np.int32)).to(eng.device)
    if last:
      flat = draw(PROMPT * PACK)
      pos = torch.arange(PROMPT, dtype=torch.int32, device=eng.device).repeat(PACK)
      starts = np.arange(PACK) * PROMPT
      packed = lambda: eng.prefill_concat(params=params, padded_tokens=flat, decoder_positions=pos, decoder_segment_ids=None, start_pos=starts, true_lengths=[PROMPT] * PACK, num_prompts=PACK)
      packed()
      dt = _best(packed)
      out["prefill_packed"] = {"tokens": PROMPT * PACK, "ms": dt * 1e3, "tokens_per_s": PROMPT * PACK / dt}
      long_ = draw(LONG)

      def chunked():
        done, pre = 0, None
        while done < LONG:
          old = None if done == 0 else maxengine.ExistingPrefix(cache=pre["cache"], common_prefix_tokens=long_[:done])
          pre, _ = eng.prefill(params=params, padded_tokens=long_[done:done + CHUNK], true_length=CHUNK, slot=0, existing_prefix=old)
          done += CHUNK
        eng.release_pages(0)

      chunked()
      dt = _best(chunked)
      out["prefill_long"] = {"tokens": LONG, "chunk": CHUNK, "ms": dt * 1e3, "tokens_per_s": LONG / dt}
      log(f"prefill {out}")
    state = eng.init_decode_state()
    prompt = draw(CONTEXT)
    pre, _ = eng.prefill(params=params, padded_tokens=prompt, true_length=CONTEXT, slot=0)
    state = eng.bulk_insert(pre, state, list(range(slots)))
    for _ in range(3):
      state, _ = eng.generate(params, state)

    def steps():
      nonlocal state
      for _ in range(8):
        state, _ = eng.generate(params, state)

    dt = _best(steps) / 8
    out[f"decode_{slots}"] = {"ms_per_step": dt * 1e3, "tokens_per_s": slots / dt}
    log(f"decode {slots}: {dt * 1e3:.3f} ms")
    eng.close()
    del eng
    torch.cuda.empty_cache()
  return out


def run(args) -> int:
  from . import build, pyconfig  # pylint: disable=import-outside-toplevel
  import sys  # pylint: disable=import-outside-toplevel
  base = os.path.join(pyconfig.PKG_DIR, "configs", "base.yml")
  names = list(SIZES) if args.hybrid == "all" else args.hybrid.split(",")
  log = lambda m: print(f"[hybrid] {m}", file=sys.stderr, flush=True)
  slots_list = [8, 128]
  rows = {}
  for name in names:
    cfg_json, like = SIZES[name]
    design = cfg_json["architecture"].lower()
    common = lambda slots: dict(attention="paged", scan_layers=False, per_device_batch_size=float(slots), max_prefill_predict_length=CHUNK, max_target_length=LONG + 32,
                                pagedattn_tokens_per_page=32, pagedattn_num_pages=2 + max(slots * 34, LONG // 32 + 2 + PACK * PROMPT // 32 + 8), use_chunked_prefill=True,
                                ixt_staging_groups=PACK, ixt_max_packed_rows=PROMPT * PACK, run_name="bench", ixt_use_hip_graph=not args.no_graph)
    with tempfile.TemporaryDirectory() as d:
      with open(os.path.join(d, "config.json"), "w", encoding="utf-8") as f:
        json.dump(cfg_json, f)
      mine = _measure(lambda slots: pyconfig.initialize(["bench", base], ixt_model_dir=d, **common(slots)), slots_list, args.opt, lambda m: log(f"{name} {design} {m}"))
    closest = _measure(lambda slots: pyconfig.initialize(["bench", base], vocab_size=32000, head_dim=128, **like, **common(slots)), slots_list, args.opt,
                       lambda m: log(f"{name} closest {m}"))
    time_of = lambda r: r.get("ms", r.get("ms_per_step"))
    rows[name] = {design: mine, "closest": closest, "closest_model": like.get("decoder_block", "llama2"), "time_ratio": {k: time_of(mine[k]) / time_of(closest[k]) for k in mine}}
  print(json.dumps({"metric": "hybrid_decoder_rates", "data": "synthetic", "dtype": "bf16", "build_id": build.source_hash(), "rows": rows}), flush=True)
  return 0
