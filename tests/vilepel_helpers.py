"""Small Vilepel models for the tests: config dicts, random weights (bf16 values), engines on model folders, comparisons with vilepel_ref."""
import json
import os

import numpy as np
import torch
from safetensors.torch import save_file

import helpers as H
import vilepel_ref as V


def latent(heads=3, dim=24, rot=16, vdim=20, rank=40, window=11, base=3000.0, scale=0.2):
  return {"type": "latent_attention", "mixer": {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "kv_rank": rank, "scale": scale,
                                                "mask": {"size": window}, "rot": {"base": base, "dims": rot}}}


def delta(heads=6, kv_heads=3, dim=20, vdim=12, conv=4):
  return {"type": "channel_delta", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}}


def dense(ff=72, limit=1.5):
  return {"kind": "dense", "ff": ff, "limit": limit}


def moe(ff=40, limit=1.25, experts=5, top=3):
  return {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "router": {"experts": experts, "top": top}}


def model(layers, vocab=203, width=88, eps=3e-5, scale=2.5):
  return {"architecture": "Vilepel", "embedding": {"scale": scale}, "norm": {"eps": eps}, "vocab": vocab, "width": width, "layers": layers}


def with_mlp(layer, mlp, weights_of=None):
  out = dict(layer, mlp=mlp)
  if weights_of is not None:
    out["weights_of"] = weights_of
  return out


def mixed_model(**kw):
  """Every kind of layer, shared weights both ways round, a layer without feed-forward; no two sizes alike."""
  a, d = latent(), delta()
  b = latent(heads=5, dim=12, rot=6, vdim=28, rank=72, window=19, base=500.0, scale=0.3)
  return model([with_mlp(d, moe()), with_mlp(a, dense()), with_mlp(b, moe(ff=24, experts=7, top=2)), with_mlp(a, dense(), weights_of=1), with_mlp(d, moe(), weights_of=0),
                with_mlp(delta(heads=4, kv_heads=4, dim=36, vdim=17, conv=2), None)], **kw)


def random_weights(cfg, seed=0, decay_rank=10, gate_rank=7):
  """{name: float64 array of bf16 values}."""
  rng = np.random.default_rng(seed)
  E = cfg["width"]
  shapes = {"embed": (cfg["vocab"], E), "final.norm": (E,), "head": (cfg["vocab"], E)}
  for i, l in enumerate(cfg["layers"]):
    if l.get("weights_of") is not None:
      continue
    m, p = l["mixer"], f"l{i}."
    shapes[p + "norm1"] = (E,)
    Hn = m["heads"]
    if l["type"] == "latent_attention":
      shapes.update({p + "mix.q": (Hn * (m["dim"] + m["rot_dim"]), E), p + "mix.dkv": (m["kv_rank"] + m["rot_dim"], E), p + "mix.dkv.norm": (m["kv_rank"],),
                     p + "mix.uk": (Hn * m["dim"], m["kv_rank"]), p + "mix.uv": (Hn * m["vdim"], m["kv_rank"]), p + "mix.o": (E, Hn * m["vdim"])})
    else:
      kd, vd = m["kv_heads"] * m["dim"], Hn * m["vdim"]
      for t, n in (("q", kd), ("k", kd), ("v", vd)):
        shapes[p + f"mix.{t}"], shapes[p + f"mix.{t}.conv"] = (n, E), (n, m["conv"])
      shapes.update({p + "mix.b": (Hn, E), p + "mix.A_log": (Hn,), p + "mix.norm": (m["vdim"],), p + "mix.a1": (decay_rank, E), p + "mix.a2": (Hn * m["dim"], decay_rank),
                     p + "mix.dt_bias": (Hn * m["dim"],), p + "mix.g1": (gate_rank, E), p + "mix.g2": (vd, gate_rank), p + "mix.o": (E, vd)})
    f = l.get("mlp")
    if f is None:
      continue
    shapes[p + "norm2"] = (E,)
    n = f["ff"] if f["kind"] == "dense" else f["expert"]["ff"]
    for q in (["mlp."] if f["kind"] == "dense" else [f"mlp.e{e}." for e in range(f["router"]["experts"])]):
      shapes.update({p + q + "gate": (n, E), p + q + "up": (n, E), p + q + "down": (E, n)})
    if f["kind"] == "moe":
      shapes[p + "mlp.router"] = (f["router"]["experts"], E)
  out = {}
  for name, shape in shapes.items():
    z = rng.standard_normal(shape)
    leaf = name.rsplit(".", 1)[-1]
    if name == "final.norm" or leaf in ("norm1", "norm2"):
      z *= 0.3
    elif leaf == "norm":
      z = 1.0 + 0.3 * z
    elif leaf == "A_log":
      z = 0.7 * z - 1.0
    elif leaf == "dt_bias":
      z = z - 1.0
    elif leaf == "conv":
      z /= np.sqrt(shape[1])
    elif name == "embed":
      z *= 3.0 / cfg["embedding"]["scale"]    # a stream well above what a sublayer adds: rounding is not blown up from layer to layer
    elif leaf == "router":
      z *= 1.5 / np.sqrt(shape[1])
    elif leaf in ("gate", "up"):
      z *= 0.6 / np.sqrt(shape[1])          # far enough for the clamps to act
    else:
      z /= np.sqrt(shape[-1])
    out[name] = torch.from_numpy(z).to(torch.bfloat16).to(torch.float64).numpy()
  return out


def write_model(path, cfg, weights):
  os.makedirs(path, exist_ok=True)
  with open(os.path.join(path, "config.json"), "w", encoding="utf-8") as f:
    json.dump(cfg, f)
  save_file({k: torch.from_numpy(np.array(v, order="C")).to(torch.bfloat16) for k, v in weights.items()}, os.path.join(path, "model.safetensors"))
  return str(path)


def config(path, dtype="float32", slots=4, pages=16, page=8, target=96, rows=96, **kw):
  return H.pyconfig.initialize(["test", H.BASE_YML], ixt_model_dir=str(path), dtype=dtype, attention="paged", scan_layers=False, per_device_batch_size=float(slots),
                               max_target_length=target, max_prefill_predict_length=rows, pagedattn_tokens_per_page=page, pagedattn_num_pages=pages + 1,
                               use_chunked_prefill=True, enable_checkpointing=False, run_name="test", **kw)


def engine(path, **kw):
  eng = H.maxengine_module().MaxEngine(config(path, **kw))
  return eng, eng.load_params()


def tokens(cfg, n, seed):
  return np.random.default_rng(seed).integers(0, cfg["vocab"], n).astype(np.int32)


def rel(got, want):
  """Per position: rms of the difference of the centred logits over the rms of the expected ones (all positions)."""
  got, want = np.asarray(got, np.float64), np.asarray(want, np.float64)
  d = got - want
  d -= d.mean(axis=-1, keepdims=True)
  scale = np.sqrt(np.mean((want - want.mean(axis=-1, keepdims=True)) ** 2))
  return np.sqrt(np.mean(d * d, axis=-1)) / scale


# one sequence's error against the float64 restatement: f32 sees rounding of a few hundred terms per sum; bf16 rounds every operand (rounding the
# restatement's own linear inputs to bf16 gives a 0.9 quantile of 0.015 to 0.018 on the mixed model)
TOL = {"float32": 3e-5, "bfloat16": 0.03}


def check(got, want, dtype, what=""):
  r = rel(got, want)
  if dtype == "float32":
    assert r.max() < TOL[dtype], (what, int(r.argmax()), r.max())
  else:                 # a routing decision can be close: one expert for another at a few positions is rounding, not a fault
    assert np.quantile(r, 0.9) < TOL[dtype] * (1 if r.size >= 10 else 3), (what, np.quantile(r, 0.9), r.max())


def scheduler(eng):
  import importlib
  return importlib.import_module("maxtext-indextts2_amd.inference.step_scheduler").StepScheduler(eng)


def run_portions(sched, rid, toks, cuts):
  """All logits of one request fed in portions; cuts = portion sizes, the last one repeated."""
  out, at, i = [], 0, 0
  while at < len(toks):
    n = min(cuts[min(i, len(cuts) - 1)], len(toks) - at)
    lg, _ = sched.step([(rid, toks[at:at + n], list(range(n)))])
    out.append(lg.cpu().numpy())
    at, i = at + n, i + 1
  return np.concatenate(out)
