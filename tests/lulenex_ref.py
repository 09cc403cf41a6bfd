"""Plain restatement of the Lulenex decoder in float64 numpy: one function per mechanism, one sequence at a time, no cache.

Used by the tests only.  Nothing here is shared with the product; every formula is written out from the equations in the docstrings.
A model is (config dict, {tensor name: float64 array}); linear weights are [out, in]."""
import numpy as np

from suzulix_ref import layer_runs, retention_states, rotate_halves
from vilepel_ref import linear, rms, sigmoid, silu, softplus, under


def one_number_norm(x, g, eps):
  """x / sqrt(mean(x^2) + eps) g, g a single number."""
  return rms(x, eps) * g


def token_shift(h, mu):
  """h_t + (h_(t-1) - h_t) mu feature by feature, with h_(-1) = 0."""
  before = np.concatenate([np.zeros_like(h[:1]), h[:-1]])
  return h + (before - h) * mu


def enter_pass(x, x0, w_in, step):
  """In front of a pass: W [x; x0] + step."""
  return linear(w_in, np.concatenate([x, x0], axis=-1)) + step


def short_convolution(x, taps, bias):
  """x [T, channels]: y_t = sum_j taps[:, j] x_(t - n + 1 + j) + bias, zeros before the start."""
  n = taps.shape[1]
  padded = np.concatenate([np.zeros((n - 1, x.shape[1])), x])
  return sum(padded[j:j + x.shape[0]] * taps[:, j] for j in range(n)) + bias


def selective_scan(x, dt, A, B, C, D):
  """x, dt [T, channels], A [channels, states], B, C [T, states]: S <- exp(dt A) S + dt x B, y = S C + D x, from zero."""
  S, y = np.zeros_like(A), np.empty_like(x)
  for t in range(x.shape[0]):
    S = np.exp(dt[t][:, None] * A) * S + (dt[t] * x[t])[:, None] * B[t][None, :]
    y[t] = S @ C[t] + D * x[t]
  return y


def mamba(h, w, m, eps):
  n, r, s = m["inner"], m["dt_rank"], m["state"]
  both = linear(w["in"], h)
  x = silu(short_convolution(both[:, :n], w["conv"], w["conv.b"]))
  low = linear(w["x"], x)
  dt = softplus(linear(w["dt"], low[:, :r]) + w["dt.b"])
  y = selective_scan(x, dt, -np.exp(w["A_log"]), low[:, r:r + s], low[:, r + s:], w["D"])
  return linear(w["o"], y * silu(both[:, n:]))


def seen(T, size):
  """[i, j]: key j at or before i and in the same chunk of `size` positions (None: no chunks)."""
  i, j = np.arange(T)[:, None], np.arange(T)[None, :]
  return (j <= i) & (True if size is None else i // size == j // size)


def sink_softmax(scores, mask, sink):
  """exp(s_ij) / (exp(sink) + sum of exp(s_ik) over the visible k), zero where the mask is."""
  s = np.where(mask, scores, -np.inf)
  top = np.maximum(s.max(axis=1, keepdims=True), sink)
  e = np.exp(s - top)
  return e / (e.sum(axis=1, keepdims=True) + np.exp(sink - top))


def chunked_attention(h, w, m, eps):
  """Keys are their own values; rotated queries and keys over their root mean square; one gate per head."""
  T, H, G, d = h.shape[0], m["heads"], m["kv_heads"], m["dim"]
  pos = np.arange(T, dtype=np.float64)
  q = (linear(w["q"], h) + w["q.b"]).reshape(T, H, d)
  k = (linear(w["k"], h) + w["k.b"]).reshape(T, G, d)
  gate = sigmoid(linear(w["g"], h))
  mask = seen(T, (m.get("mask") or {}).get("size"))
  out = np.empty((T, H, d))
  for i in range(H):
    g = i // (H // G)
    s = rms(rotate_halves(q[:, i], pos, m["rot"]), eps) @ rms(rotate_halves(k[:, g], pos, m["rot"]), eps).T * m["scale"]
    out[:, i] = gate[:, i:i + 1] * (sink_softmax(s, mask, w["sink"][i]) @ k[:, g])
  return linear(w["o"], out.reshape(T, H * d)) + w["o.b"]


def lightning(h, w, m, eps):
  """silu queries, keys and values, one decay per head; the heads normed together by a plain weight, gated."""
  T, H, d, dv = h.shape[0], m["heads"], m["dim"], m["vdim"]
  q, k, v = (silu(linear(w[n], h)).reshape(T, H, -1) for n in ("q", "k", "v"))
  out = np.concatenate([retention_states(q[:, i], k[:, i], v[:, i], m["decay"][i]) for i in range(H)], axis=1)
  return linear(w["o"], rms(out, eps) * w["norm"] * sigmoid(linear(w["g"], h)))


def parallel(h, w, m, eps):
  return m["left_scale"] * chunked_attention(h, under(w, "left."), m["left"], eps) + m["right_scale"] * lightning(h, under(w, "right."), m["right"], eps)


MIXERS = {"mamba1": mamba, "parallel": parallel}


def xielu(z, p, q):
  """softplus(p) z^2 + z / 2 for z > 0, (1/2 + softplus(q)) (exp(z) - 1 - z) + z / 2 for the others."""
  low = np.minimum(z, 0.0)
  return np.where(z > 0, softplus(p) * z * z, (0.5 + softplus(q)) * (np.expm1(low) - low)) + 0.5 * z


def unit(h, w):
  return linear(w["down"], xielu(linear(w["up"], h), *w["act"]))


def pass_starts(config):
  """{place among the layer runs: number of the pass that begins there}."""
  loop = config.get("loop")
  return {loop["start"] + t * (loop["stop"] - loop["start"]): t for t in range(loop["times"])} if loop else {}


def forward(config, weights, tokens, taps=None):
  """Logits [T, vocab] of one token sequence; `taps` (a list) collects the residual stream after every layer run."""
  eps = config["norm"]["eps"]
  x = x0 = weights["embed"][np.asarray(tokens)]
  starts = pass_starts(config)
  for run, i in enumerate(layer_runs(config)):
    if run in starts:
      x = enter_pass(x, x0, weights["loop.in"], weights["loop.step"][starts[run]])
    layer, p = config["layers"][i], f"l{i}."
    h = token_shift(one_number_norm(x, weights[p + "norm1"], eps), weights[p + "shift"])
    x = x + MIXERS[layer["type"]](h, under(weights, p + "mix."), layer["mixer"], eps)
    if layer.get("mlp") is not None:
      x = x + unit(one_number_norm(x, weights[p + "norm2"], eps), under(weights, p + "mlp."))
    if taps is not None:
      taps.append(x)
  return linear(weights["head"], one_number_norm(x, weights["final.norm"], eps))
