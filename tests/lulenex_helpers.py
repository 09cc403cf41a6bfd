"""Small Lulenex models for the tests: config dicts and random weights (bf16 values).  Engines, portions and comparisons are vilepel_helpers'."""
import numpy as np
import torch

import vilepel_helpers as VH


def left(heads=6, kv_heads=3, dim=18, dims=10, base=700.0, scale=0.3, chunk=23):
  return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "rot": {"base": base, "dims": dims}, "scale": scale, "mask": None if chunk is None else {"size": chunk}}


def right(heads=3, dim=22, vdim=30, decay=None):
  return {"heads": heads, "dim": dim, "vdim": vdim, "decay": [1.0 - 2.0 ** -(2 + 1.5 * i) for i in range(heads)] if decay is None else decay}


def parallel(l=None, r=None, left_scale=0.8, right_scale=0.6):
  return {"type": "parallel", "mixer": {"left": left() if l is None else l, "right": right() if r is None else r, "left_scale": left_scale, "right_scale": right_scale}}


def mamba(inner=70, state=9, dt_rank=7, conv=3):
  return {"type": "mamba1", "mixer": {"inner": inner, "state": state, "dt_rank": dt_rank, "conv": conv}}


def dense(ff=120):
  return {"kind": "dense", "ff": ff}


def with_mlp(layer, mlp):
  return dict(layer, mlp=mlp)


def model(layers, vocab=203, width=88, eps=3e-5, loop=None):
  return {"architecture": "Lulenex", "norm": {"eps": eps}, "vocab": vocab, "width": width, "loop": loop, "layers": layers}


def mixed_model(**kw):
  """Every kind of layer, no two sizes alike, a loop in the middle, a layer without a feed-forward."""
  return model([with_mlp(mamba(), dense()), with_mlp(parallel(), dense(ff=75)), with_mlp(mamba(inner=130, state=20, dt_rank=11, conv=4), None),
                with_mlp(parallel(left(heads=4, kv_heads=1, dim=30, dims=30, base=5000.0, scale=0.2, chunk=16), right(heads=2, dim=34, vdim=18, decay=[0.5, 0.9990234375]), 1.1, 0.4),
                         dense(ff=33)),
                with_mlp(parallel(left(heads=2, kv_heads=2, dim=24, dims=6, chunk=None), right(heads=5, dim=8, vdim=12)), dense(ff=200))],
               **dict(dict(loop={"start": 1, "stop": 4, "times": 2}), **kw))


def shapes(cfg):
  E = cfg["width"]
  out = {"embed": (cfg["vocab"], E), "final.norm": (), "head": (cfg["vocab"], E)}
  if cfg["loop"]:
    out.update({"loop.in": (E, 2 * E), "loop.step": (cfg["loop"]["times"], E)})
  for i, layer in enumerate(cfg["layers"]):
    m, p = layer["mixer"], f"l{i}."
    out.update({p + "norm1": (), p + "shift": (E,)})
    if layer["type"] == "mamba1":
      C, N, r = m["inner"], m["state"], m["dt_rank"]
      out.update({p + "mix.in": (2 * C, E), p + "mix.conv": (C, m["conv"]), p + "mix.conv.b": (C,), p + "mix.x": (r + 2 * N, C), p + "mix.dt": (C, r), p + "mix.dt.b": (C,),
                  p + "mix.A_log": (C, N), p + "mix.D": (C,), p + "mix.o": (E, C)})
    else:
      a, b = m["left"], m["right"]
      H, G, d = a["heads"], a["kv_heads"], a["dim"]
      for t, n in (("q", H * d), ("k", G * d)):
        out.update({p + f"mix.left.{t}": (n, E), p + f"mix.left.{t}.b": (n,)})
      out.update({p + "mix.left.sink": (H,), p + "mix.left.g": (H, E), p + "mix.left.o": (E, H * d), p + "mix.left.o.b": (E,)})
      kq, v = b["heads"] * b["dim"], b["heads"] * b["vdim"]
      out.update({p + "mix.right.q": (kq, E), p + "mix.right.k": (kq, E), p + "mix.right.v": (v, E), p + "mix.right.g": (v, E), p + "mix.right.norm": (v,), p + "mix.right.o": (E, v)})
    if layer["mlp"] is not None:
      n = layer["mlp"]["ff"]
      out.update({p + "norm2": (), p + "mlp.up": (n, E), p + "mlp.down": (E, n), p + "mlp.act": (2,)})
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
      z = 3.0 * z                      # a stream well above what a sublayer adds: rounding is not blown up from layer to layer
    elif leaf in ("norm1", "norm2", "norm") or name == "final.norm":
      z = 1.0 + 0.3 * z
    elif leaf == "shift":
      z = 0.5 + 0.4 * z
    elif leaf == "A_log":
      z = 0.8 * z - 0.5
    elif name.endswith("dt.b"):
      z = 0.8 * z - 1.0
    elif leaf == "D":
      z = 1.0 + 0.4 * z
    elif leaf == "sink":
      z = 1.0 + z
    elif leaf == "b":
      z = 0.4 * z
    elif leaf == "act":
      z = 0.7 * z
    elif leaf == "step":
      z = 0.7 * z
    elif leaf == "conv":
      z = z / np.sqrt(shape[1])
    elif name == "loop.in":            # about as large as its inputs
      z = z / np.sqrt(shape[1] / 2)
    else:
      z = z / np.sqrt(shape[-1])
    out[name] = np.asarray(z)
  return rounded(out)


# f32 sees rounding of a few hundred terms per sum, bf16 the rounding of every operand: rounding the restatement's own linear inputs alone gives a 0.9
# quantile of 0.0035 to 0.0041 on the mixed model
TOL = {"float32": 3e-5, "bfloat16": 0.012}
rel = VH.rel


def check(got, want, dtype, what=""):
  r = rel(got, want)
  if dtype == "float32":
    assert r.max() < TOL[dtype], (what, int(r.argmax()), r.max())
  else:
    assert np.quantile(r, 0.9) < TOL[dtype] * (1 if r.size >= 10 else 2) and r.max() < 3 * TOL[dtype], (what, np.quantile(r, 0.9), r.max())
