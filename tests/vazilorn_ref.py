"""Plain restatement of the Vazilorn decoder in float64 numpy: one function per mechanism, one sequence at a time, no cache.

Used by the tests only.  Nothing here is shared with the product; every formula is written out from the equations in the docstrings.
A model is (config dict, {tensor name: float64 array}); linear weights are [out, in]."""
import numpy as np

from vilepel_ref import linear, rms, sigmoid, silu, under


def tanh_norm(x, alpha, w, b):
  """y = w tanh(alpha x) + b, feature by feature (alpha a scalar): no statistic of x enters."""
  return np.tanh(alpha * x) * w + b


def gelu_tanh(z):
  """z / 2 (1 + tanh(sqrt(2 / pi) (z + 0.044715 z^3)))."""
  return 0.5 * z * (1.0 + np.tanh(np.sqrt(2.0 / np.pi) * (z + 0.044715 * z ** 3)))


def gated_unit(h, wg, wu, wd, act):
  return linear(wd, act(linear(wg, h)) * linear(wu, h))


def frequencies(dims, base, scaling):
  """Turning rate of plane i: base^(-2 i / dims), stretched by its wavelength l = 2 pi / f: unchanged below original / high, divided by `factor` above
  original / low, in between the mixture whose share of the unchanged rate is (original / l - low) / (high - low)."""
  out = []
  for i in range(dims // 2):
    f = base ** (-2.0 * i / dims)
    if scaling is not None:
      l = 2.0 * np.pi / f
      if l > scaling["original"] / scaling["low"]:
        f = f / scaling["factor"]
      elif l >= scaling["original"] / scaling["high"]:
        s = (scaling["original"] / l - scaling["low"]) / (scaling["high"] - scaling["low"])
        f = s * f + (1.0 - s) * f / scaling["factor"]
    out.append(f)
  return np.array(out)


def rotate_first(x, pos, rot):
  """x [T, dim]: the first rot.dims features turn in planes of neighbours (2 i, 2 i + 1), the others stay."""
  n = rot["dims"]
  a = pos[:, None] * frequencies(n, rot["base"], rot.get("scaling"))[None, :]
  c, s = np.cos(a), np.sin(a)
  y = x.copy()
  y[:, 0:n:2] = x[:, 0:n:2] * c - x[:, 1:n:2] * s
  y[:, 1:n:2] = x[:, 1:n:2] * c + x[:, 0:n:2] * s
  return y


def sink_softmax(scores, window, sink):
  """Row i over columns i - window + 1 .. i: exp(s_ij) / (sum_j exp(s_ij) + exp(sink))."""
  T = scores.shape[0]
  i, j = np.arange(T)[:, None], np.arange(T)[None, :]
  s = np.where((i - j >= 0) & (i - j < window), scores, -np.inf)
  m = np.maximum(s.max(axis=1, keepdims=True), sink)
  e = np.exp(s - m)
  return e / (e.sum(axis=1, keepdims=True) + np.exp(sink - m))


def attention(h, w, m, eps):
  """h [T, width]; w: the mixer's tensors by short name; m: the mixer's sizes."""
  T = h.shape[0]
  H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
  pos = np.arange(T, dtype=np.float64)
  q = rms(linear(w["q"], h).reshape(T, H, d), eps) * w["q.norm"]
  k = rms(linear(w["k"], h).reshape(T, G, d), eps) * w["k.norm"]
  v = linear(w["v"], h).reshape(T, G, dv)
  out = np.empty((T, H, dv))
  for i in range(H):
    g = i // (H // G)
    s = rotate_first(q[:, i], pos, m["rot"]) @ rotate_first(k[:, g], pos, m["rot"]).T * m["scale"]
    out[:, i] = sink_softmax(s, m["mask"]["size"], w["sink"][i]) @ v[:, g]
  return linear(w["o"], out.reshape(T, H * dv))


def route(h, router, correction, r):
  """-> per token (chosen experts, their weights).  Choice by sigmoid(z) + correction inside the groups whose two best choice scores add up to most;
  weights are the plain sigmoids, divided by their sum, times r.scale."""
  s = sigmoid(linear(router, h))
  n, count, keep = r["experts"], r["groups"]["count"], r["groups"]["keep"]
  size = n // count
  picks, weights = [], []
  for t in range(h.shape[0]):
    choice = s[t] + correction
    score = [np.sort(choice[g * size:(g + 1) * size])[-2:].sum() for g in range(count)]
    best = np.argsort(-np.array(score), kind="stable")[:keep]
    open_ = np.full(n, -np.inf)
    for g in best:
      open_[g * size:(g + 1) * size] = choice[g * size:(g + 1) * size]
    p = np.argsort(-open_, kind="stable")[:r["top"]]
    picks.append(p)
    weights.append(s[t, p] / (s[t, p].sum() + 1e-20) * r["scale"])
  return picks, weights


def mixture(h, w, m):
  picks, weights = route(h, w["router"], w["correction"], m["router"])
  out = gated_unit(h, w["shared.gate"], w["shared.up"], w["shared.down"], silu)
  for t in range(h.shape[0]):
    for e, a in zip(picks[t], weights[t]):
      out[t] += a * gated_unit(h[t:t + 1], w[f"e{e}.gate"], w[f"e{e}.up"], w[f"e{e}.down"], silu)[0]
  return out


def feed_forward(h, w, m):
  return gated_unit(h, w["gate"], w["up"], w["down"], gelu_tanh) if m["kind"] == "dense" else mixture(h, w, m)


def forward(config, weights, tokens, taps=None):
  """Logits [T, vocab] of one token sequence; `taps` (a list) collects the residual stream after every layer."""
  eps = config["norm"]["eps"]
  norm = lambda x, name: tanh_norm(x, weights[name + ".alpha"], weights[name], weights[name + ".b"])
  x = weights["embed"][np.asarray(tokens)]
  for i, layer in enumerate(config["layers"]):
    p = f"l{i}."
    x = x + norm(attention(norm(x, p + "norm1"), under(weights, p + "mix."), layer["mixer"], eps), p + "norm1b")
    if layer.get("mlp") is not None:
      x = x + norm(feed_forward(norm(x, p + "norm2"), under(weights, p + "mlp."), layer["mlp"]), p + "norm2b")
    if taps is not None:
      taps.append(x.copy())
  return linear(weights["head"], norm(x, "final.norm"))
