"""Plain restatement of the Vilepel decoder in float64 numpy: one function per mechanism, one sequence at a time, no cache.

Used by the tests only.  Nothing here is shared with the product; every formula is written out from the equations in the docstrings.
A model is (config dict, {tensor name: float64 array}); linear weights are [out, in]."""
import numpy as np


def linear(w, x):
  """y_t = W x_t for every row t of x."""
  return x @ w.T


def rms(x, eps):
  """x / sqrt(mean(x^2) + eps) over the last axis."""
  return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def zero_centred_norm(x, w, eps):
  """rms(x) (1 + w)."""
  return rms(x, eps) * (1.0 + w)


def sigmoid(z):
  return 1.0 / (1.0 + np.exp(-z))


def silu(z):
  return z * sigmoid(z)


def softplus(z):
  return np.logaddexp(0.0, z)


def rotate_pairs(x, pos, base):
  """x [..., T, dims], positions pos [T]: features 2i and 2i + 1 form a plane that turns by p base^(-2i/dims)."""
  dims = x.shape[-1]
  f = base ** (-np.arange(0, dims, 2) / dims)
  a = pos[:, None] * f[None, :]
  c, s = np.cos(a), np.sin(a)
  u, v = x[..., 0::2], x[..., 1::2]
  y = np.empty_like(x)
  y[..., 0::2] = u * c - v * s
  y[..., 1::2] = v * c + u * s
  return y


def window_softmax(scores, window):
  """scores [T, T] -> softmax weights of row i over columns i - window + 1 .. i."""
  T = scores.shape[0]
  i, j = np.arange(T)[:, None], np.arange(T)[None, :]
  s = np.where((i - j >= 0) & (i - j < window), scores, -np.inf)
  e = np.exp(s - s.max(axis=1, keepdims=True))
  return e / e.sum(axis=1, keepdims=True)


def latent_attention(h, w, m, eps):
  """h [T, width]; w: the mixer's tensors by short name; m: the mixer's sizes."""
  T = h.shape[0]
  H, dn, dr, dv, rank = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
  pos = np.arange(T, dtype=np.float64)
  q = linear(w["q"], h).reshape(T, H, dn + dr)
  d = linear(w["dkv"], h)
  c = rms(d[:, :rank], eps) * w["dkv.norm"]
  kr = rotate_pairs(d[:, rank:], pos, m["rot"]["base"])
  ku = linear(w["uk"], c).reshape(T, H, dn)
  v = linear(w["uv"], c).reshape(T, H, dv)
  out = np.empty((T, H, dv))
  for i in range(H):
    qr = rotate_pairs(q[:, i, dn:], pos, m["rot"]["base"])
    s = (q[:, i, :dn] @ ku[:, i].T + qr @ kr.T) * m["scale"]
    out[:, i] = window_softmax(s, m["mask"]["size"]) @ v[:, i]
  return linear(w["o"], out.reshape(T, H * dv))


def short_conv(x, taps):
  """x [T, channels], taps [channels, n] -> y_t = sum_b taps[:, n - 1 - b] x_{t - b}, with x_{<0} = 0."""
  n = taps.shape[1]
  padded = np.concatenate([np.zeros((n - 1, x.shape[1])), x])
  return sum(padded[j:j + x.shape[0]] * taps[:, j] for j in range(n))


def unit(x):
  return x / np.sqrt(np.sum(x * x, axis=-1, keepdims=True) + 1e-6)


def delta_rule(q, k, v, g, beta):
  """One head: q, k, g [T, dim], v [T, vdim], beta [T] -> o [T, vdim].  S (dim x vdim) starts at zero."""
  S = np.zeros((q.shape[1], v.shape[1]))
  o = np.empty_like(v)
  for t in range(q.shape[0]):
    S = g[t][:, None] * S
    u = beta[t] * (v[t] - S.T @ k[t])
    S = S + np.outer(k[t], u)
    o[t] = S.T @ q[t]
  return o


def channel_delta(h, w, m, eps):
  T = h.shape[0]
  H, KH, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
  q = silu(short_conv(linear(w["q"], h), w["q.conv"])).reshape(T, KH, d)
  k = silu(short_conv(linear(w["k"], h), w["k.conv"])).reshape(T, KH, d)
  v = silu(short_conv(linear(w["v"], h), w["v.conv"])).reshape(T, H, dv)
  q, k = unit(q) * d ** -0.5, unit(k)
  beta = sigmoid(linear(w["b"], h))
  a = linear(w["a2"], linear(w["a1"], h)) + w["dt_bias"]
  g = np.exp(-np.exp(w["A_log"])[None, :, None] * softplus(a).reshape(T, H, d))
  gate = sigmoid(linear(w["g2"], linear(w["g1"], h))).reshape(T, H, dv)
  o = np.empty((T, H, dv))
  for i in range(H):
    j = i // (H // KH)
    o[:, i] = delta_rule(q[:, j], k[:, j], v[:, i], g[:, i], beta[:, i])
  o = rms(o, eps) * w["norm"] * gate
  return linear(w["o"], o.reshape(T, H * dv))


def clamped_glu(h, wg, wu, wd, limit):
  g = np.minimum(linear(wg, h), limit)
  u = np.clip(linear(wu, h), -limit, limit)
  return linear(wd, g * sigmoid(1.702 * g) * (u + 1.0))


def route(h, router, top):
  """-> (experts [T, top] by descending softmax probability, those probabilities)."""
  z = linear(router, h)
  e = np.exp(z - z.max(axis=1, keepdims=True))
  s = e / e.sum(axis=1, keepdims=True)
  idx = np.argsort(-s, axis=1, kind="stable")[:, :top]
  return idx, np.take_along_axis(s, idx, axis=1)


def mixture(h, w, m):
  idx, s = route(h, w["router"], m["router"]["top"])
  out = np.zeros_like(h)
  for t in range(h.shape[0]):
    for j, e in enumerate(idx[t]):
      out[t] += s[t, j] * clamped_glu(h[t:t + 1], w[f"e{e}.gate"], w[f"e{e}.up"], w[f"e{e}.down"], m["expert"]["limit"])[0]
  return out


def feed_forward(h, w, m):
  return clamped_glu(h, w["gate"], w["up"], w["down"], m["limit"]) if m["kind"] == "dense" else mixture(h, w, m)


MIXERS = {"latent_attention": latent_attention, "channel_delta": channel_delta}


def under(weights, prefix):
  return {k[len(prefix):]: v for k, v in weights.items() if k.startswith(prefix)}


def forward(config, weights, tokens, taps=None):
  """Logits [T, vocab] of one token sequence; `taps` (a list) collects the residual stream after every layer."""
  eps = config["norm"]["eps"]
  x = weights["embed"][np.asarray(tokens)] * config["embedding"]["scale"]
  for i, layer in enumerate(config["layers"]):
    p = f"l{layer.get('weights_of', i)}."
    x = x + zero_centred_norm(MIXERS[layer["type"]](x, under(weights, p + "mix."), layer["mixer"], eps), weights[p + "norm1"], eps)
    if layer.get("mlp") is not None:
      x = x + zero_centred_norm(feed_forward(x, under(weights, p + "mlp."), layer["mlp"]), weights[p + "norm2"], eps)
    if taps is not None:
      taps.append(x.copy())
  return linear(weights["head"], zero_centred_norm(x, weights["final.norm"], eps))
