"""Plain restatement of the Suzulix decoder in float64 numpy: one function per mechanism, one sequence at a time, no cache.

Used by the tests only.  Nothing here is shared with the product; every formula is written out from the equations in the docstrings.
A model is (config dict, {tensor name: float64 array}); linear weights are [out, in]."""
import numpy as np

from vilepel_ref import linear, rms, sigmoid, silu, under


def layer_norm(x, w, b, eps):
  """(x - mean) / sqrt(mean((x - mean)^2) + eps) w + b over the last axis."""
  c = x - x.mean(axis=-1, keepdims=True)
  return c / np.sqrt(np.mean(c * c, axis=-1, keepdims=True) + eps) * w + b


def angles(pos, rot):
  """[T, dims / 2]: plane i turns by p base^(-2 i / dims)."""
  n = rot["dims"]
  return pos[:, None] * rot["base"] ** (-2.0 * np.arange(n // 2) / n)[None, :]


def rotate_neighbours(x, pos, rot):
  """x [T, dim]: the first rot.dims features turn in planes (2 i, 2 i + 1), the others stay."""
  n, a = rot["dims"], angles(pos, rot)
  y = x.copy()
  y[:, 0:n:2] = x[:, 0:n:2] * np.cos(a) - x[:, 1:n:2] * np.sin(a)
  y[:, 1:n:2] = x[:, 1:n:2] * np.cos(a) + x[:, 0:n:2] * np.sin(a)
  return y


def rotate_halves(x, pos, rot):
  """x [T, dim]: the first rot.dims features turn in planes (i, i + dims / 2), the others stay."""
  n, h, a = rot["dims"], rot["dims"] // 2, angles(pos, rot)
  y = x.copy()
  y[:, :h] = x[:, :h] * np.cos(a) - x[:, h:n] * np.sin(a)
  y[:, h:n] = x[:, h:n] * np.cos(a) + x[:, :h] * np.sin(a)
  return y


def causal_softmax(scores):
  """Row i over columns 0 .. i."""
  T = scores.shape[0]
  s = np.where(np.tril(np.ones((T, T), bool)), scores, -np.inf)
  e = np.exp(s - s.max(axis=1, keepdims=True))
  return e / e.sum(axis=1, keepdims=True)


def capped(s, cap):
  return cap * np.tanh(s / cap)


def latent_attention(h, w, m, eps):
  """Queries by way of a normed latent; keys and values are up-projections of a normed latent plus one rotated key part for all heads; gated heads."""
  T, H, d, r, dv = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"]
  pos = np.arange(T, dtype=np.float64)
  q = linear(w["uq"], rms(linear(w["dq"], h), eps) * w["dq.norm"]).reshape(T, H, d + r)
  low = linear(w["dkv"], h)
  c = rms(low[:, :m["kv_rank"]], eps) * w["dkv.norm"]
  kr = rotate_halves(low[:, m["kv_rank"]:], pos, m["rot"])
  k, v = linear(w["uk"], c).reshape(T, H, d), linear(w["uv"], c).reshape(T, H, dv)
  out = np.empty((T, H, dv))
  for i in range(H):
    s = q[:, i, :d] @ k[:, i].T + rotate_halves(q[:, i, d:], pos, m["rot"]) @ kr.T
    out[:, i] = causal_softmax(s * m["scale"]) @ v[:, i]
  return linear(w["o"], out.reshape(T, H * dv) * sigmoid(linear(w["g"], h)))


def mixing_factor(w, diff):
  """lambda = exp(lq1 . lk1) - exp(lq2 . lk2) + diff."""
  return np.exp(np.sum(w["lq1"] * w["lk1"])) - np.exp(np.sum(w["lq2"] * w["lk2"])) + diff


def differential_attention(h, w, m, eps):
  """Two softmax maps per head over the same values; a1 - lambda a2, normed per head, times 1 - diff, gated."""
  T, H, G, d, dv = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
  pos = np.arange(T, dtype=np.float64)
  q, k, v = linear(w["q"], h).reshape(T, H, 2, d), linear(w["k"], h).reshape(T, G, 2, d), linear(w["v"], h).reshape(T, G, dv)
  lam = mixing_factor(w, m["diff"])
  out = np.empty((T, H, dv))
  for i in range(H):
    g = i // (H // G)
    a = [causal_softmax(capped(rotate_neighbours(q[:, i, j], pos, m["rot"]) @ rotate_neighbours(k[:, g, j], pos, m["rot"]).T * m["scale"], m["softcap"])) @ v[:, g] for j in range(2)]
    out[:, i] = rms(a[0] - lam * a[1], eps) * (1.0 - m["diff"])
  return linear(w["o"], out.reshape(T, H * dv) * sigmoid(linear(w["g"], h)))


def retention_states(q, k, v, decay):
  """S_t = decay S_(t-1) + k_t v_t^T from zero, o_t = S_t^T q_t."""
  S, out = np.zeros((k.shape[1], v.shape[1])), np.empty_like(v)
  for t in range(k.shape[0]):
    S = decay * S + np.outer(k[t], v[t])
    out[t] = S.T @ q[t]
  return out


def retention(h, w, m, eps):
  T, H, d, dv = h.shape[0], m["heads"], m["dim"], m["vdim"]
  pos = np.arange(T, dtype=np.float64)
  q, k, v = linear(w["q"], h).reshape(T, H, d), linear(w["k"], h).reshape(T, H, d), linear(w["v"], h).reshape(T, H, dv)
  out = np.empty((T, H, dv))
  for i in range(H):
    out[:, i] = rms(retention_states(rotate_halves(q[:, i], pos, m["rot"]), rotate_halves(k[:, i], pos, m["rot"]) * d ** -0.5, v[:, i], m["decay"][i]), eps)
  return linear(w["o"], out.reshape(T, H * dv) * silu(linear(w["g"], h)))


MIXERS = {"latent_attention": latent_attention, "attention": differential_attention, "retention": retention}


def square_unit(h, up, down):
  """down relu(up h)^2."""
  return linear(down, np.maximum(linear(up, h), 0.0) ** 2)


def route(h, router, bias, top):
  """-> per token (chosen experts, softmax over their logits)."""
  z = linear(router, h) + bias
  picks = np.argsort(-z, axis=1, kind="stable")[:, :top]
  c = np.take_along_axis(z, picks, axis=1)
  e = np.exp(c - c.max(axis=1, keepdims=True))
  return picks, e / e.sum(axis=1, keepdims=True)


def mixture(h, w, m):
  picks, weights = route(h, w["router"], w["router.b"], m["router"]["top"])
  out = np.zeros_like(h)
  if m.get("shared"):
    out += sigmoid(linear(w["shared.sg"], h)) * square_unit(h, w["shared.up"], w["shared.down"])
  for t in range(h.shape[0]):
    for e, a in zip(picks[t], weights[t]):
      out[t] += a * square_unit(h[t:t + 1], w[f"e{e}.up"], w[f"e{e}.down"])[0]
  return out


def gather_streams(x, w):
  """x [T, streams, width] -> sum_s in[s] x_s."""
  return np.einsum("tse,s->te", x, w["in"])


def spread_streams(x, y, w):
  """x_t <- sum_s mix[s, t] x_s + out[t] y."""
  return np.einsum("tse,su->tue", x, w["mix"]) + w["out"][None, :, None] * y[:, None, :]


def layer_runs(config):
  """Layers in the order they run: loop.start .. stop - 1 `times` times in a row, then the rest."""
  n, loop = len(config["layers"]), config.get("loop")
  if not loop:
    return list(range(n))
  body = list(range(loop["start"], loop["stop"]))
  return list(range(loop["start"])) + body * loop["times"] + list(range(loop["stop"], n))


def forward(config, weights, tokens, taps=None):
  """Logits [T, vocab] of one token sequence; `taps` (a list) collects the sum of the streams after every layer run."""
  eps = config["norm"]["eps"]
  norm = lambda x, name: layer_norm(x, weights[name], weights[name + ".b"], eps)
  x = np.repeat((weights["embed"][np.asarray(tokens)] * config["embedding"]["scale"])[:, None, :], config["streams"], axis=1)
  for i in layer_runs(config):
    layer, p = config["layers"][i], f"l{i}."
    hc = under(weights, p + "hc1.")
    x = spread_streams(x, MIXERS[layer["type"]](norm(gather_streams(x, hc), p + "norm1"), under(weights, p + "mix."), layer["mixer"], eps), hc)
    if layer.get("mlp") is not None:
      hc = under(weights, p + "hc2.")
      x = spread_streams(x, mixture(norm(gather_streams(x, hc), p + "norm2"), under(weights, p + "mlp."), layer["mlp"]), hc)
    if taps is not None:
      taps.append(x.sum(axis=1))
  return linear(weights["embed"], norm(x.sum(axis=1), "final.norm")) * config["logit_scale"]
