"""Small Vazilorn models for the tests: config dicts and random weights (bf16 values).  Engines, portions and comparisons are vilepel_helpers'."""
import numpy as np
import torch

import vilepel_helpers as VH

SCALING = {"factor": 4.0, "low": 1.0, "high": 4.0, "original": 40}      # all three regimes inside a short test


def attn(heads=6, kv_heads=3, dim=24, vdim=20, window=11, base=300.0, dims=16, scale=0.25, scaling=SCALING):
  return {"type": "attention", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "mask": {"size": window},
                                         "rot": {"base": base, "dims": dims, "scaling": scaling}}}


def dense(ff=72):
  return {"kind": "dense", "ff": ff}


def moe(ff=40, experts=6, top=3, groups=3, keep=2, scale=1.7, shared=56):
  return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top, "groups": {"count": groups, "keep": keep}, "scale": scale}, "shared": {"ff": shared}}


def model(layers, vocab=203, width=88, eps=3e-5):
  return {"architecture": "Vazilorn", "norm": {"eps": eps}, "vocab": vocab, "width": width, "layers": layers}


def with_mlp(layer, mlp):
  return dict(layer, mlp=mlp)


def mixed_model(**kw):
  """Dense, routed and missing feed-forwards on attention layers of which no two are alike."""
  return model([with_mlp(attn(), dense()), with_mlp(attn(heads=5, kv_heads=1, dim=40, vdim=12, window=19, base=900.0, dims=6, scale=0.2, scaling=None), moe()),
                with_mlp(attn(heads=4, kv_heads=4, dim=18, vdim=36, window=33, dims=18, scale=0.3), None),
                with_mlp(attn(heads=4, kv_heads=2, dim=12, vdim=28, window=7, dims=4, scale=0.4, base=50.0), moe(ff=24, experts=8, top=2, groups=4, keep=1, scale=0.6, shared=200)),
                with_mlp(attn(window=26), dense(40))], **kw)


def random_weights(cfg, seed=0):
  """{name: float64 array of bf16 values}."""
  rng = np.random.default_rng(seed)
  E = cfg["width"]
  shapes = {"embed": (cfg["vocab"], E), "head": (cfg["vocab"], E)}

  def norm(name):
    shapes.update({name: (E,), name + ".b": (E,), name + ".alpha": ()})

  def gated(name, n):
    shapes.update({name + "gate": (n, E), name + "up": (n, E), name + "down": (E, n)})

  norm("final.norm")
  for i, l in enumerate(cfg["layers"]):
    m, p = l["mixer"], f"l{i}."
    for n in ("norm1", "norm1b", "norm2", "norm2b"):
      norm(p + n)
    shapes.update({p + "mix.q": (m["heads"] * m["dim"], E), p + "mix.k": (m["kv_heads"] * m["dim"], E), p + "mix.v": (m["kv_heads"] * m["vdim"], E), p + "mix.sink": (m["heads"],),
                   p + "mix.q.norm": (m["dim"],), p + "mix.k.norm": (m["dim"],), p + "mix.o": (E, m["heads"] * m["vdim"])})
    f = l.get("mlp")
    if f is not None and f["kind"] == "dense":
      gated(p + "mlp.", f["ff"])
    elif f is not None:
      for e in range(f["router"]["experts"]):
        gated(p + f"mlp.e{e}.", f["expert"]["ff"])
      gated(p + "mlp.shared.", f["shared"]["ff"])
      shapes.update({p + "mlp.router": (f["router"]["experts"], E), p + "mlp.correction": (f["router"]["experts"],)})
  out = {}
  for name, shape in shapes.items():
    z = rng.standard_normal(shape)
    leaf = name.rsplit(".", 1)[-1]
    if leaf == "alpha":
      z = (2.5 if "1b." in name or "2b." in name else 0.6) + 0.1 * z     # what a sublayer adds is as large as the stream
    elif leaf == "b":
      z = 0.1 * z
    elif leaf in ("norm", "norm1", "norm1b", "norm2", "norm2b"):
      z = 1.0 + 0.3 * z
    elif leaf == "sink":
      z = 1.5 + z
    elif leaf == "correction":
      z = 0.2 * z - 0.5
    elif name == "embed":
      z *= 1.5
    elif leaf == "router":
      z *= 3.0 / np.sqrt(shape[1])
    else:
      z /= np.sqrt(shape[-1])
    out[name] = torch.from_numpy(np.asarray(z)).to(torch.bfloat16).to(torch.float64).numpy()
  return out


def rounded(w):
  """The nearest bf16 values."""
  return {k: torch.from_numpy(np.asarray(v)).to(torch.bfloat16).to(torch.float64).numpy() for k, v in w.items()}


# as for Vilepel: f32 sees rounding of a few hundred terms per sum, bf16 the rounding of every linear input
TOL = VH.TOL
check, rel = VH.check, VH.rel
