"""Model folders (config.json + model.safetensors) -> the engine's configuration keys.

`read_model_dir` looks the folder's `architecture` up in ARCHITECTURES; a reader turns config.json (and, for sizes that only a tensor's shape
tells, the safetensors header) into config keys: vocabulary and width, `decoder_block: hybrid` and one HybridLayer per layer (include/ixt.h,
ixt_layer).  A new design of known mechanisms needs a reader here and nothing else."""
from __future__ import annotations

import dataclasses
import json
import os
import struct
from typing import Any, Callable, Dict, Mapping, Optional, Sequence, Tuple

MIX_LATENT_ATTENTION, MIX_GATED_DELTA, MIX_ATTENTION, MIX_RETENTION, MIX_LIGHTNING, MIX_SCAN = 0, 1, 2, 3, 4, 5
RECURRENT_MIXERS = (MIX_GATED_DELTA, MIX_RETENTION, MIX_LIGHTNING, MIX_SCAN)
FFN_NONE, FFN_DENSE, FFN_MOE = 0, 1, 2
GLU_CLAMPED, GLU_GELU_TANH, GLU_SILU, ACT_RELU2, ACT_XIELU = 1, 2, 3, 4, 5      # from ACT_RELU2 on: no gate
ROUTE_SOFTMAX, ROUTE_SIGMOID, ROUTE_CHOSEN = 0, 1, 2
ROPE_NEIGHBOURS, ROPE_HALVES = 0, 1
NORM_RMS, NORM_TANH, NORM_LAYER, NORM_ONE = 0, 1, 2, 3
GATE_FEATURES, GATE_HEADS = 1, 2
QK_NORM_WEIGHTS, QK_NORM_PLAIN = 1, 2
NORM_BEFORE, NORM_AFTER = 1, 2


@dataclasses.dataclass(frozen=True)
class HybridLayer:
  """One layer of a hybrid decoder; the fields of ixt_layer."""
  mixer: int
  weights_of: int = -1
  heads: int = 1
  dim: int = 1
  vdim: int = 1
  rot_dim: int = 0
  kv_rank: int = 0
  window: int = 0
  rope_base: float = 10000.0
  attn_scale: float = 1.0
  kv_heads: int = 1
  conv: int = 1
  decay_rank: int = 1
  gate_rank: int = 1
  ffn: int = FFN_NONE
  ff: int = 0
  glu_limit: float = 0.0
  experts: int = 0
  top: int = 0
  qk_norm: int = 0
  sink: int = 0
  rope_factor: float = 0.0
  rope_low: float = 1.0
  rope_high: float = 1.0
  rope_original: float = 1.0
  glu: int = GLU_CLAMPED
  router: int = ROUTE_SOFTMAX
  router_correction: int = 0
  groups: int = 1
  groups_keep: int = 1
  router_norm: int = 0
  router_scale: float = 1.0
  shared_ff: int = 0
  number: int = -1
  rope_pairs: int = ROPE_NEIGHBOURS
  q_rank: int = 0
  out_gate: int = 0
  maps: int = 1
  map_diff: float = 0.0
  softcap: float = 0.0
  router_bias: int = 0
  shared_gate: int = 0
  decay: Tuple[float, ...] = ()
  chunk: int = 0
  key_values: int = 0
  mix_bias: int = 0
  inner: int = 1
  state: int = 1
  dt_rank: int = 1
  mix_scale: float = 1.0
  beside: Optional["HybridLayer"] = None
  shift: int = 0
  loop_pass: int = -1


def carries_state(l: HybridLayer) -> bool:
  """The layer has more than a cache of keys: tokens must come in order, and a run cannot start over in the middle."""
  return l.mixer in RECURRENT_MIXERS or bool(l.shift) or (l.beside is not None and carries_state(l.beside))


Shapes = Mapping[str, Tuple[int, ...]]


def safetensors_shapes(path: str) -> Dict[str, Tuple[int, ...]]:
  """{tensor name: shape} from the header of a safetensors file (8-byte little-endian length, then JSON)."""
  with open(path, "rb") as f:
    (n,) = struct.unpack("<Q", f.read(8))
    header = json.loads(f.read(n))
  return {k: tuple(v["shape"]) for k, v in header.items() if k != "__metadata__"}


def _vilepel_feed_forward(mlp: Any) -> Dict[str, Any]:
  if mlp is None:
    return {"ffn": FFN_NONE}
  if mlp["kind"] == "dense":
    return {"ffn": FFN_DENSE, "ff": int(mlp["ff"]), "glu_limit": float(mlp["limit"])}
  if mlp["kind"] == "moe":
    return {"ffn": FFN_MOE, "ff": int(mlp["expert"]["ff"]), "glu_limit": float(mlp["expert"]["limit"]),
            "experts": int(mlp["router"]["experts"]), "top": int(mlp["router"]["top"])}
  raise ValueError(f"Vilepel: feed-forward kind {mlp['kind']!r}")


def _vilepel_latent(m: Mapping[str, Any], name: Callable[[str], str], shapes: Shapes) -> Dict[str, Any]:
  del name, shapes
  rot = m["rot"]
  if int(rot["dims"]) != int(m["rot_dim"]):
    raise ValueError(f"Vilepel: rot.dims ({rot['dims']}) must equal rot_dim ({m['rot_dim']})")
  return {"mixer": MIX_LATENT_ATTENTION, "heads": int(m["heads"]), "dim": int(m["dim"]), "vdim": int(m["vdim"]), "rot_dim": int(m["rot_dim"]),
          "kv_rank": int(m["kv_rank"]), "window": int((m.get("mask") or {}).get("size") or 0), "rope_base": float(rot["base"]), "attn_scale": float(m["scale"])}


def _vilepel_delta(m: Mapping[str, Any], name: Callable[[str], str], shapes: Shapes) -> Dict[str, Any]:
  # config.json does not give the two ranks: a1 is [decay rank, width], g1 [gate rank, width].  Without weights (synthetic ones): the key dims.
  rank = lambda t: int(shapes[name(t)][0]) if name(t) in shapes else int(m["dim"])
  return {"mixer": MIX_GATED_DELTA, "heads": int(m["heads"]), "kv_heads": int(m["kv_heads"]), "dim": int(m["dim"]), "vdim": int(m["vdim"]), "conv": int(m["conv"]),
          "decay_rank": rank("a1"), "gate_rank": rank("g1")}


_VILEPEL_MIXERS = {"latent_attention": _vilepel_latent, "channel_delta": _vilepel_delta}


def vilepel_keys(cfg: Mapping[str, Any], shapes: Shapes) -> Dict[str, Any]:
  """Vilepel: latent-attention and gated-delta layers in any order, zero-centred RMS norms behind every sublayer, clamped gated units (dense or routed)."""
  layers = []
  for i, entry in enumerate(cfg["layers"]):
    src = entry.get("weights_of")
    src = -1 if src is None else int(src)
    if entry["type"] not in _VILEPEL_MIXERS:
      raise ValueError(f"Vilepel: layer {i} has type {entry['type']!r}")
    own = i if src < 0 else src
    spec = _VILEPEL_MIXERS[entry["type"]](entry["mixer"], lambda t, own=own: f"l{own}.mix.{t}", shapes)
    layers.append(HybridLayer(weights_of=src, **spec, **_vilepel_feed_forward(entry.get("mlp"))))
  return {
      "decoder_block": "hybrid",
      "vocab_size": int(cfg["vocab"]),
      "base_emb_dim": int(cfg["width"]),
      "base_num_decoder_layers": len(layers),
      "normalization_layer_epsilon": float(cfg["norm"]["eps"]),
      "embedding_scale": float(cfg["embedding"]["scale"]),
      "hybrid_layers": tuple(layers),
  }


def _vazilorn_mixer(m: Mapping[str, Any]) -> Dict[str, Any]:
  rot = m["rot"]
  heads, kv_heads, dim, dims = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(rot["dims"])
  if heads % kv_heads or dims % 2 or dims > dim:
    raise ValueError(f"Vazilorn: {heads} heads over {kv_heads} key heads, {dims} of {dim} dims rotated")
  out = {"mixer": MIX_ATTENTION, "heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": int(m["vdim"]), "rot_dim": dims, "rope_base": float(rot["base"]),
         "window": int((m.get("mask") or {}).get("size") or 0), "attn_scale": float(m["scale"]), "qk_norm": 1, "sink": 1}
  scaling = rot.get("scaling")
  if scaling:
    out.update(rope_factor=float(scaling["factor"]), rope_low=float(scaling["low"]), rope_high=float(scaling["high"]), rope_original=float(scaling["original"]))
  return out


def _vazilorn_feed_forward(mlp: Any) -> Dict[str, Any]:
  if mlp is None:
    return {"ffn": FFN_NONE}
  if mlp["kind"] == "dense":
    return {"ffn": FFN_DENSE, "ff": int(mlp["ff"]), "glu": GLU_GELU_TANH}
  if mlp["kind"] == "moe":
    r, groups, shared = mlp["router"], mlp["router"].get("groups") or {}, mlp.get("shared") or {}
    return {"ffn": FFN_MOE, "ff": int(mlp["expert"]["ff"]), "glu": GLU_SILU, "experts": int(r["experts"]), "top": int(r["top"]), "router": ROUTE_SIGMOID,
            "router_correction": 1, "groups": int(groups.get("count") or 1), "groups_keep": int(groups.get("keep") or 1), "router_norm": 1,
            "router_scale": float(r["scale"]), "shared_ff": int(shared.get("ff") or 0)}
  raise ValueError(f"Vazilorn: feed-forward kind {mlp['kind']!r}")


def vazilorn_keys(cfg: Mapping[str, Any], shapes: Shapes) -> Dict[str, Any]:
  """Vazilorn: windowed attention with sinks, normed queries and keys and scaled rotations; tanh norms on both sides of every sublayer; gelu units or a
  routed mixture of silu units (sigmoid scores, groups, a shared unit)."""
  del shapes
  layers = []
  for i, entry in enumerate(cfg["layers"]):
    if entry["type"] != "attention":
      raise ValueError(f"Vazilorn: layer {i} has type {entry['type']!r}")
    layers.append(HybridLayer(**_vazilorn_mixer(entry["mixer"]), **_vazilorn_feed_forward(entry.get("mlp"))))
  return {
      "decoder_block": "hybrid",
      "vocab_size": int(cfg["vocab"]),
      "base_emb_dim": int(cfg["width"]),
      "base_num_decoder_layers": len(layers),
      "normalization_layer_epsilon": float(cfg["norm"]["eps"]),
      "hybrid_norm_kind": NORM_TANH,
      "hybrid_norm_places": NORM_BEFORE | NORM_AFTER,
      "hybrid_layers": tuple(layers),
  }


def _suzulix_latent(m: Mapping[str, Any]) -> Dict[str, Any]:
  rot = m["rot"]
  if int(rot["dims"]) != int(m["rot_dim"]):
    raise ValueError(f"Suzulix: rot.dims ({rot['dims']}) must equal rot_dim ({m['rot_dim']})")
  return {"mixer": MIX_LATENT_ATTENTION, "heads": int(m["heads"]), "dim": int(m["dim"]), "vdim": int(m["vdim"]), "rot_dim": int(m["rot_dim"]), "kv_rank": int(m["kv_rank"]),
          "q_rank": int(m["q_rank"]), "rope_base": float(rot["base"]), "rope_pairs": ROPE_HALVES, "attn_scale": float(m["scale"]), "out_gate": 1}


def _suzulix_attention(m: Mapping[str, Any]) -> Dict[str, Any]:
  rot = m["rot"]
  heads, kv_heads, dim, dims = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(rot["dims"])
  if heads % kv_heads or dims % 2 or dims > dim:
    raise ValueError(f"Suzulix: {heads} heads over {kv_heads} key heads, {dims} of {dim} dims rotated")
  return {"mixer": MIX_ATTENTION, "heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": int(m["vdim"]), "rot_dim": dims, "rope_base": float(rot["base"]),
          "attn_scale": float(m["scale"]), "softcap": float(m["softcap"]), "maps": 2, "map_diff": float(m["diff"]), "out_gate": 1}


def _suzulix_retention(m: Mapping[str, Any]) -> Dict[str, Any]:
  rot, decay = m["rot"], tuple(float(d) for d in m["decay"])
  heads, dim, dims = int(m["heads"]), int(m["dim"]), int(rot["dims"])
  if len(decay) != heads or dims % 2 or dims > dim:
    raise ValueError(f"Suzulix: {len(decay)} decays for {heads} heads, {dims} of {dim} dims rotated")
  return {"mixer": MIX_RETENTION, "heads": heads, "dim": dim, "vdim": int(m["vdim"]), "rot_dim": dims, "rope_base": float(rot["base"]), "rope_pairs": ROPE_HALVES, "decay": decay}


_SUZULIX_MIXERS = {"latent_attention": _suzulix_latent, "attention": _suzulix_attention, "retention": _suzulix_retention}


def _suzulix_feed_forward(mlp: Any) -> Dict[str, Any]:
  if mlp is None:
    return {"ffn": FFN_NONE}
  if mlp["kind"] != "moe":
    raise ValueError(f"Suzulix: feed-forward kind {mlp['kind']!r}")
  shared = mlp.get("shared") or {}
  return {"ffn": FFN_MOE, "ff": int(mlp["expert"]["ff"]), "glu": ACT_RELU2, "experts": int(mlp["router"]["experts"]), "top": int(mlp["router"]["top"]), "router": ROUTE_CHOSEN,
          "router_bias": 1, "shared_ff": int(shared.get("ff") or 0), "shared_gate": 1 if shared.get("ff") else 0}


def suzulix_keys(cfg: Mapping[str, Any], shapes: Shapes) -> Dict[str, Any]:
  """Suzulix: latent attention, differential attention and retention in any order, a stretch of layers run several times; layer norms in front,
  hyper-connections, routed squared-relu units with a gated shared one, the embedding table as the head."""
  del shapes
  layers = []
  for i, entry in enumerate(cfg["layers"]):
    if entry["type"] not in _SUZULIX_MIXERS:
      raise ValueError(f"Suzulix: layer {i} has type {entry['type']!r}")
    layers.append(HybridLayer(number=i, **_SUZULIX_MIXERS[entry["type"]](entry["mixer"]), **_suzulix_feed_forward(entry.get("mlp"))))
  loop = cfg.get("loop")
  return {
      "decoder_block": "hybrid",
      "vocab_size": int(cfg["vocab"]),
      "base_emb_dim": int(cfg["width"]),
      "normalization_layer_epsilon": float(cfg["norm"]["eps"]),
      "embedding_scale": float(cfg["embedding"]["scale"]),
      "logits_via_embedding": True,
      "logit_scale": float(cfg["logit_scale"]),
      "hybrid_norm_kind": NORM_LAYER,
      "hybrid_norm_places": NORM_BEFORE,
      "hybrid_streams": int(cfg["streams"]),
      **_looped(layers, *((int(loop["start"]), int(loop["stop"]), int(loop["times"])) if loop else (0, 0, 1))),
  }


def _lulenex_attention(m: Mapping[str, Any], factor: float) -> Dict[str, Any]:
  rot = m["rot"]
  heads, kv_heads, dim, dims = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(rot["dims"])
  if heads % kv_heads or dims % 2 or dims > dim:
    raise ValueError(f"Lulenex: {heads} heads over {kv_heads} key heads, {dims} of {dim} dims rotated")
  if int(m["vdim"]) != dim:
    raise ValueError(f"Lulenex: the values are the keys, vdim ({m['vdim']}) must equal dim ({dim})")
  return {"mixer": MIX_ATTENTION, "heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "rot_dim": dims, "rope_base": float(rot["base"]), "rope_pairs": ROPE_HALVES,
          "chunk": int((m.get("mask") or {}).get("size") or 0), "attn_scale": float(m["scale"]), "qk_norm": QK_NORM_PLAIN, "sink": 1, "out_gate": GATE_HEADS, "key_values": 1, "mix_bias": 1,
          "mix_scale": factor}


def _lulenex_lightning(m: Mapping[str, Any], factor: float) -> HybridLayer:
  decay = tuple(float(d) for d in m["decay"])
  if len(decay) != int(m["heads"]):
    raise ValueError(f"Lulenex: {len(decay)} decays for {m['heads']} heads")
  return HybridLayer(mixer=MIX_LIGHTNING, heads=int(m["heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]), decay=decay, mix_scale=factor)


def _lulenex_parallel(m: Mapping[str, Any]) -> Dict[str, Any]:
  return dict(_lulenex_attention(m["left"], float(m["left_scale"])), beside=_lulenex_lightning(m["right"], float(m["right_scale"])))


def _lulenex_scan(m: Mapping[str, Any]) -> Dict[str, Any]:
  return {"mixer": MIX_SCAN, "inner": int(m["inner"]), "state": int(m["state"]), "dt_rank": int(m["dt_rank"]), "conv": int(m["conv"])}


_LULENEX_MIXERS = {"parallel": _lulenex_parallel, "mamba1": _lulenex_scan}


def _lulenex_feed_forward(mlp: Any) -> Dict[str, Any]:
  if mlp is None:
    return {"ffn": FFN_NONE}
  if mlp["kind"] != "dense":
    raise ValueError(f"Lulenex: feed-forward kind {mlp['kind']!r}")
  return {"ffn": FFN_DENSE, "ff": int(mlp["ff"]), "glu": ACT_XIELU}


def lulenex_keys(cfg: Mapping[str, Any], shapes: Shapes) -> Dict[str, Any]:
  """Lulenex: chunked attention beside lightning attention, or a selective scan, in any order behind one-number norms and a token shift; xIELU units; a
  stretch of layers run several times, the embedding output joining in front of every pass."""
  del shapes
  layers = []
  for i, entry in enumerate(cfg["layers"]):
    if entry["type"] not in _LULENEX_MIXERS:
      raise ValueError(f"Lulenex: layer {i} has type {entry['type']!r}")
    layers.append(HybridLayer(number=i, shift=1, **_LULENEX_MIXERS[entry["type"]](entry["mixer"]), **_lulenex_feed_forward(entry.get("mlp"))))
  loop = cfg.get("loop")
  keys = _looped(layers, *((int(loop["start"]), int(loop["stop"]), int(loop["times"])) if loop else (0, 0, 1)))
  if loop and int(loop["stop"]) > int(loop["start"]):
    runs, start, span = list(keys["hybrid_layers"]), int(loop["start"]), int(loop["stop"]) - int(loop["start"])
    for t in range(int(loop["times"])):
      runs[start + t * span] = dataclasses.replace(runs[start + t * span], loop_pass=t)
    keys["hybrid_layers"] = tuple(runs)
  return {
      "decoder_block": "hybrid",
      "vocab_size": int(cfg["vocab"]),
      "base_emb_dim": int(cfg["width"]),
      "normalization_layer_epsilon": float(cfg["norm"]["eps"]),
      "hybrid_norm_kind": NORM_ONE,
      "hybrid_norm_places": NORM_BEFORE,
      **keys,
  }


def _looped(layers: Sequence[HybridLayer], start: int, stop: int, times: int) -> Dict[str, Any]:
  """Layers start .. stop - 1 `times` times in a row: every further pass is a run of its own (cache, state) on the first one's parameters."""
  if not 0 <= start <= stop <= len(layers) or times < 1:
    raise ValueError(f"loop {start} .. {stop}, {times} times, over {len(layers)} layers")
  again = [dataclasses.replace(layers[i], weights_of=i) for _ in range(times - 1) for i in range(start, stop)]
  runs = tuple(layers[:stop]) + tuple(again) + tuple(layers[stop:])
  return {"base_num_decoder_layers": len(runs), "hybrid_layers": runs}


ARCHITECTURES: Dict[str, Callable[[Mapping[str, Any], Shapes], Dict[str, Any]]] = {
    "Lulenex": lulenex_keys,
    "Suzulix": suzulix_keys,
    "Vazilorn": vazilorn_keys,
    "Vilepel": vilepel_keys,
}


def read_model_dir(path: str) -> Dict[str, Any]:
  """Config keys of the model in `path`; `load_parameters_path` names its weights when they are there."""
  with open(os.path.join(path, "config.json"), "r", encoding="utf-8") as f:
    cfg = json.load(f)
  name = cfg.get("architecture")
  if name not in ARCHITECTURES:
    raise ValueError(f"{path}: architecture {name!r} is not built (built: {sorted(ARCHITECTURES)})")
  weights = os.path.join(path, "model.safetensors")
  have = os.path.isfile(weights)
  keys = ARCHITECTURES[name](cfg, safetensors_shapes(weights) if have else {})
  if have:
    keys["load_parameters_path"] = weights
  return keys


def parameter_shapes(config: Any) -> Dict[str, Tuple[int, ...]]:
  """{tensor name: shape} of a hybrid decoder; linear weights are [out, in]."""
  E, V, S = int(config.emb_dim), int(config.vocab_size), int(config.hybrid_streams)
  out: Dict[str, Tuple[int, ...]] = {"embed": (V, E)}
  if not config.logits_via_embedding:
    out["head"] = (V, E)

  def norm(name: str) -> None:
    out[name] = () if config.hybrid_norm_kind == NORM_ONE else (E,)
    if config.hybrid_norm_kind in (NORM_TANH, NORM_LAYER):
      out[name + ".b"] = (E,)
    if config.hybrid_norm_kind == NORM_TANH:
      out[name + ".alpha"] = ()

  def unit(name: str, ff: int, kind: int) -> None:
    if kind < ACT_RELU2:
      out[name + "gate"] = (ff, E)
    out[name + "up"], out[name + "down"] = (ff, E), (E, ff)

  both = config.hybrid_norm_places == NORM_BEFORE | NORM_AFTER
  norm("final.norm")
  passes = 1 + max(l.loop_pass for l in config.hybrid_layers)
  if passes > 0:
    out["loop.in"], out["loop.step"] = (E, 2 * E), (passes, E)

  def attention(p: str, l: HybridLayer) -> None:
    sizes = {"q": l.heads * l.maps * l.dim, "k": l.kv_heads * l.maps * l.dim}
    if not l.key_values:
      sizes["v"] = l.kv_heads * l.vdim
    out.update({p + t: (n, E) for t, n in sizes.items()})
    out[p + "o"] = (E, l.heads * l.vdim)
    if l.mix_bias:
      out.update({p + t + ".b": (n,) for t, n in dict(sizes, o=E).items()})
    if l.maps > 1:
      out.update({p + n: (l.dim,) for n in ("lq1", "lk1", "lq2", "lk2")})
    if l.qk_norm == QK_NORM_WEIGHTS:
      out[p + "q.norm"] = out[p + "k.norm"] = (l.dim,)
    if l.sink:
      out[p + "sink"] = (l.heads,)
    if l.out_gate:
      out[p + "g"] = (l.heads * (l.vdim if l.out_gate == GATE_FEATURES else 1), E)

  def linear_attention(p: str, l: HybridLayer) -> None:
    kq, v = l.heads * l.dim, l.heads * l.vdim
    out.update({p + "q": (kq, E), p + "k": (kq, E), p + "v": (v, E), p + "g": (v, E), p + "o": (E, v)})
    if l.mixer == MIX_LIGHTNING:
      out[p + "norm"] = (v,)

  for i, l in enumerate(config.hybrid_layers):
    if l.weights_of >= 0:
      continue
    p = f"l{i if l.number < 0 else l.number}."
    for q in ("hc1.", "hc2.")[:0 if S == 0 else 1 if l.ffn == FFN_NONE else 2]:
      out.update({p + q + "in": (S,), p + q + "out": (S,), p + q + "mix": (S, S)})
    for n in ("norm1", "norm1b")[:1 + both] + (() if l.ffn == FFN_NONE else ("norm2", "norm2b")[:1 + both]):
      norm(p + n)
    if l.mixer == MIX_LATENT_ATTENTION:
      if l.q_rank > 0:
        out.update({p + "mix.dq": (l.q_rank, E), p + "mix.dq.norm": (l.q_rank,), p + "mix.uq": (l.heads * (l.dim + l.rot_dim), l.q_rank)})
      else:
        out[p + "mix.q"] = (l.heads * (l.dim + l.rot_dim), E)
      out.update({p + "mix.dkv": (l.kv_rank + l.rot_dim, E), p + "mix.dkv.norm": (l.kv_rank,),
                  p + "mix.uk": (l.heads * l.dim, l.kv_rank), p + "mix.uv": (l.heads * l.vdim, l.kv_rank), p + "mix.o": (E, l.heads * l.vdim)})
      if l.out_gate:
        out[p + "mix.g"] = (l.heads * l.vdim, E)
    elif l.mixer in (MIX_ATTENTION, MIX_RETENTION, MIX_LIGHTNING):
      for q, x in (("mix.", l),) if l.beside is None else (("mix.left.", l), ("mix.right.", l.beside)):
        (attention if x.mixer == MIX_ATTENTION else linear_attention)(p + q, x)
    elif l.mixer == MIX_SCAN:
      C, N, r = l.inner, l.state, l.dt_rank
      out.update({p + "mix.in": (2 * C, E), p + "mix.conv": (C, l.conv), p + "mix.conv.b": (C,), p + "mix.x": (r + 2 * N, C), p + "mix.dt": (C, r), p + "mix.dt.b": (C,),
                  p + "mix.A_log": (C, N), p + "mix.D": (C,), p + "mix.o": (E, C)})
    else:
      kq, v = l.kv_heads * l.dim, l.heads * l.vdim
      for t, n in (("q", kq), ("k", kq), ("v", v)):
        out[p + f"mix.{t}"], out[p + f"mix.{t}.conv"] = (n, E), (n, l.conv)
      out.update({p + "mix.b": (l.heads, E), p + "mix.A_log": (l.heads,), p + "mix.norm": (l.vdim,), p + "mix.a1": (l.decay_rank, E),
                  p + "mix.a2": (l.heads * l.dim, l.decay_rank), p + "mix.dt_bias": (l.heads * l.dim,), p + "mix.g1": (l.gate_rank, E),
                  p + "mix.g2": (v, l.gate_rank), p + "mix.o": (E, v)})
    if l.shift:
      out[p + "shift"] = (E,)
    if l.ffn == FFN_DENSE:
      if l.glu == ACT_XIELU:
        out[p + "mlp.act"] = (2,)
      unit(p + "mlp.", l.ff, l.glu)
    elif l.ffn == FFN_MOE:
      for e in range(l.experts):
        unit(p + f"mlp.e{e}.", l.ff, l.glu)
      out[p + "mlp.router"] = (l.experts, E)
      if l.router_bias:
        out[p + "mlp.router.b"] = (l.experts,)
      if l.router_correction:
        out[p + "mlp.correction"] = (l.experts,)
      if l.shared_ff > 0:
        unit(p + "mlp.shared.", l.shared_ff, l.glu)
        if l.shared_gate:
          out[p + "mlp.shared.sg"] = (1, E)
  return out
