"""Small Suzulix models for the tests: config dicts and random weights (bf16 values).  Engines, portions and comparisons are vilepel_helpers'."""
import numpy as np
import torch

import vilepel_helpers as VH


def latent(heads=3, dim=20, rot=12, vdim=28, rank=44, q_rank=36, base=3000.0, scale=0.2):
  return {"type": "latent_attention", "mixer": {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "kv_rank": rank, "q_rank": q_rank, "scale": scale,
                                                "rot": {"base": base, "dims": rot}}}


def attn(heads=6, kv_heads=3, dim=18, vdim=40, dims=10, base=700.0, scale=0.3, softcap=6.0, diff=0.35):
  return {"type": "attention", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "softcap": softcap, "diff": diff,
                                         "rot": {"base": base, "dims": dims}}}


def retention(heads=3, dim=22, vdim=30, dims=14, base=400.0, decay=None):
  decay = [1.0 - 2.0 ** -(3 + 1.5 * i) for i in range(heads)] if decay is None else decay
  return {"type": "retention", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": decay, "rot": {"base": base, "dims": dims}}}


def moe(ff=40, experts=5, top=3, shared=56):
  out = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}
  return dict(out, shared={"ff": shared}) if shared else out


def with_mlp(layer, mlp):
  return dict(layer, mlp=mlp)


def model(layers, vocab=203, width=88, eps=3e-5, scale=2.5, streams=3, loop=None, logit_scale=1.5):
  return {"architecture": "Suzulix", "embedding": {"scale": scale}, "norm": {"eps": eps}, "vocab": vocab, "width": width, "streams": streams, "loop": loop,
          "logit_scale": logit_scale, "layers": layers}


def mixed_model(**kw):
  """Every kind of layer, no two sizes alike, a loop in the middle, layers without a feed-forward and without a shared unit."""
  return model([with_mlp(latent(), moe()), with_mlp(retention(), moe(ff=24, experts=7, top=2, shared=0)), with_mlp(attn(), None),
                with_mlp(attn(heads=4, kv_heads=1, dim=30, vdim=24, dims=30, softcap=15.0, diff=0.6), moe(ff=16, experts=4, top=1, shared=140)),
                with_mlp(retention(heads=2, dim=34, vdim=18, dims=34, decay=[0.5, 0.9990234375]), None),
                with_mlp(latent(heads=5, dim=12, rot=6, vdim=16, rank=72, q_rank=20, base=90.0, scale=0.3), moe(ff=33, experts=3, top=3))],
               loop={"start": 1, "stop": 4, "times": 2}, **kw)


def shapes(cfg):
  E, S = cfg["width"], cfg["streams"]
  out = {"embed": (cfg["vocab"], E), "final.norm": (E,), "final.norm.b": (E,)}
  for i, l in enumerate(cfg["layers"]):
    m, p = l["mixer"], f"l{i}."
    H, d, dv = m["heads"], m["dim"], m["vdim"]
    for q in ("1", "2")[:1 if l["mlp"] is None else 2]:
      out.update({p + "norm" + q: (E,), p + "norm" + q + ".b": (E,), p + f"hc{q}.in": (S,), p + f"hc{q}.out": (S,), p + f"hc{q}.mix": (S, S)})
    if l["type"] == "latent_attention":
      r, kv, qr = m["rot_dim"], m["kv_rank"], m["q_rank"]
      out.update({p + "mix.dq": (qr, E), p + "mix.dq.norm": (qr,), p + "mix.uq": (H * (d + r), qr), p + "mix.dkv": (kv + r, E), p + "mix.dkv.norm": (kv,),
                  p + "mix.uk": (H * d, kv), p + "mix.uv": (H * dv, kv)})
    elif l["type"] == "attention":
      G = m["kv_heads"]
      out.update({p + "mix.q": (H * 2 * d, E), p + "mix.k": (G * 2 * d, E), p + "mix.v": (G * dv, E)})
      out.update({p + f"mix.{n}": (d,) for n in ("lq1", "lk1", "lq2", "lk2")})
    else:
      out.update({p + "mix.q": (H * d, E), p + "mix.k": (H * d, E), p + "mix.v": (H * dv, E)})
    out.update({p + "mix.g": (H * dv, E), p + "mix.o": (E, H * dv)})
    f = l["mlp"]
    if f is None:
      continue
    for e in range(f["router"]["experts"]):
      out.update({p + f"mlp.e{e}.up": (f["expert"]["ff"], E), p + f"mlp.e{e}.down": (E, f["expert"]["ff"])})
    out.update({p + "mlp.router": (f["router"]["experts"], E), p + "mlp.router.b": (f["router"]["experts"],)})
    if f.get("shared"):
      n = f["shared"]["ff"]
      out.update({p + "mlp.shared.up": (n, E), p + "mlp.shared.down": (E, n), p + "mlp.shared.sg": (1, E)})
  return out


def rounded(w):
  """The nearest bf16 values."""
  return {k: torch.from_numpy(np.array(v, order="C")).to(torch.bfloat16).to(torch.float64).numpy() for k, v in w.items()}


def random_weights(cfg, seed=0):
  """{name: float64 array of bf16 values}."""
  rng = np.random.default_rng(seed)
  out = {}
  for name, shape in shapes(cfg).items():
    z = rng.standard_normal(shape)
    leaf = name.rsplit(".", 1)[-1]
    if name == "embed":
      z *= 4.0 / cfg["embedding"]["scale"]      # a stream well above what a sublayer adds: rounding is not blown up from layer to layer
    elif ".hc" in name:           # streams that differ, mix and stay of one size
      S = cfg["streams"]
      z = (0.08 * z + 0.95 * np.eye(S) if leaf == "mix" else 0.1 * z + 1.0 / S if leaf == "in" else 0.3 * z + 1.0)
    elif leaf == "b":
      z *= 1.5 if "router" in name else 0.1
    elif leaf in ("norm", "norm1", "norm2"):
      z = 1.0 + 0.3 * z
    elif leaf in ("lq1", "lk1", "lq2", "lk2"):
      z *= 0.7 / np.sqrt(np.sqrt(shape[0]))
    elif leaf == "router":
      z *= 1.5 / np.sqrt(shape[1])
    elif leaf == "up":
      z *= 0.8 / np.sqrt(shape[1])
    else:
      z /= np.sqrt(shape[-1])
    out[name] = z
  return rounded(out)


# f32 sees rounding of a few hundred terms per sum, bf16 the rounding of every operand: rounding the restatement's own linear inputs alone gives a 0.9
# quantile of 0.003 to 0.007 on the mixed model
TOL = {"float32": 3e-5, "bfloat16": 0.02}
rel = VH.rel


def check(got, want, dtype, what=""):
  r = rel(got, want)
  if dtype == "float32":
    assert r.max() < TOL[dtype], (what, int(r.argmax()), r.max())
  else:                 # (a close choice of experts may turn over with rounding)
    assert np.quantile(r, 0.9) < TOL[dtype] * (1 if r.size >= 10 else 3), (what, np.quantile(r, 0.9), r.max())
