"""Plain, slow reading of the Didipel decoder, one function per mechanism.

Float64 on the CPU by default, one sequence at a time, recurrences stepped
token by token, no cache. It shares no code with xotorch_amd: the tests hold
the framework's layers, caches and kernels against these functions.

`w` is a mapping from checkpoint tensor names to tensors, `cfg` the raw
config.json dictionary.
"""
import math

import torch


def rms(x, eps):
  return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def norm_one_plus(x, weight, eps):
  return rms(x, eps) * (1 + weight)


def silu(x):
  return x / (1 + torch.exp(-x))


def sigmoid(x):
  return 1 / (1 + torch.exp(-x))


def softplus(x):
  return torch.log1p(torch.exp(-x.abs())) + x.clamp(min=0)


def distance_bucket(n, rows, far):
  """Bucket of a distance n >= 0: the lower half of the rows one by one, the
  upper half on a logarithmic scale that saturates at distance `far`."""
  half = rows // 2
  if n < half:
    return n
  steps = math.log(n / half) / math.log(far / half) * (rows - half)
  return min(rows - 1, half + math.floor(steps + 1e-9))


def window_attention(q, k, v, bias, scale, window):
  """q [T,H,d], k [T,G,d], v [T,G,e], bias [rows of distance, H] indexed by
  i - j. A sink of score zero without a value joins the softmax."""
  T, H, _ = q.shape
  per = H // k.shape[1]
  out = q.new_zeros(T, H, v.shape[2])
  for i in range(T):
    lo = max(0, i - window + 1)
    for h in range(H):
      g = h // per
      s = (k[lo:i + 1, g] @ q[i, h]) * scale
      s = s + torch.stack([bias[i - j, h] for j in range(lo, i + 1)])
      top = torch.clamp(s.max(), min=0)
      e = torch.exp(s - top)
      p = e / (e.sum() + torch.exp(-top))
      out[i, h] = p @ v[lo:i + 1, g]
  return out


def left_mixer(h, w, p, m, eps):
  T = h.shape[0]
  H, G, d, e = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
  q = rms(h @ w[p + "q"].T, eps) * w[p + "q.norm"]
  k = rms(h @ w[p + "k"].T, eps) * w[p + "k.norm"]
  v = h @ w[p + "v"].T
  rel = w[p + "rel"]
  window = m["mask"]["size"]
  bias = torch.stack([rel[distance_bucket(n, rel.shape[0], m["bias_max"])]
                      for n in range(min(window, T))])
  o = window_attention(q.view(T, H, d), k.view(T, G, d), v.view(T, G, e), bias, m["scale"], window)
  gate = sigmoid(h @ w[p + "g"].T)
  return (o * gate[:, :, None]).reshape(T, H * e) @ w[p + "o"].T


def causal_conv(x, taps):
  """x [T,C], taps [C,n]: the last column weighs the current token."""
  n = taps.shape[1]
  padded = torch.cat([x.new_zeros(n - 1, x.shape[1]), x])
  return sum(padded[j:j + x.shape[0]] * taps[:, j] for j in range(n))


def unit(x):
  return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def delta_scan(q, k, v, g, beta):
  """q, k [T,G,d]; v [T,H,e]; g [T,H,d]; beta [T,H]."""
  T, H, e = v.shape
  per = H // q.shape[1]
  out = torch.zeros_like(v)
  for h in range(H):
    S = v.new_zeros(q.shape[2], e)
    for t in range(T):
      kk, qq = k[t, h // per], q[t, h // per]
      S = g[t, h][:, None] * S
      u = beta[t, h] * (v[t, h] - S.T @ kk)
      S = S + torch.outer(kk, u)
      out[t, h] = S.T @ qq
  return out


def right_mixer(h, w, p, m, eps):
  T = h.shape[0]
  H, G, d, e = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
  q, k, v = (silu(causal_conv(h @ w[p + n].T, w[p + n + ".conv"])) for n in "qkv")
  q = unit(q.view(T, G, d)) * d ** -0.5
  k = unit(k.view(T, G, d))
  beta = sigmoid(h @ w[p + "b"].T)
  pre = (h @ w[p + "a1"].T @ w[p + "a2"].T + w[p + "dt_bias"]).view(T, H, d)
  g = torch.exp(-torch.exp(w[p + "A_log"])[None, :, None] * softplus(pre))
  o = delta_scan(q, k, v.view(T, H, e), g, beta)
  gate = sigmoid(h @ w[p + "g1"].T @ w[p + "g2"].T).view(T, H, e)
  return (rms(o, eps) * w[p + "norm"] * gate).reshape(T, H * e) @ w[p + "o"].T


def parallel_mixer(h, w, p, m, eps):
  left = left_mixer(h, w, p + "left.", m["left"], eps)
  right = right_mixer(h, w, p + "right.", m["right"], eps)
  return m["left_scale"] * left + m["right_scale"] * right


def wkv_scan(r, k, v, decay, u):
  """r, k, v, decay [T,H,d], u [H,d]."""
  T, H, d = r.shape
  out = torch.zeros_like(v)
  for h in range(H):
    S = v.new_zeros(d, d)
    for t in range(T):
      kv = torch.outer(k[t, h], v[t, h])
      out[t, h] = (S + u[h][:, None] * kv).T @ r[t, h]
      S = decay[t, h][:, None] * S + kv
  return out


def wkv_mixer(h, w, p, m, eps):
  T = h.shape[0]
  H, d = m["heads"], m["dim"]
  before = torch.cat([torch.zeros_like(h[:1]), h[:-1]])
  mix = {n: h + (before - h) * w[p + "mu." + n] for n in "rkvgw"}
  r, k, v = ((mix[n] @ w[p + n].T).view(T, H, d) for n in "rkv")
  gate = silu(mix["g"] @ w[p + "g"].T)
  decay = torch.exp(-torch.exp(torch.tanh(mix["w"] @ w[p + "w1"].T) @ w[p + "w2"].T + w[p + "w0"]))
  o = wkv_scan(r, k, v, decay.view(T, H, d), w[p + "u"].view(H, d))
  return (rms(o, eps).reshape(T, H * d) * w[p + "norm"] * gate) @ w[p + "o"].T


def feed_forward(h, w, p):
  return (silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


MIXERS = {"parallel": parallel_mixer, "wkv": wkv_mixer}


def forward(tokens, w, cfg, dtype=torch.float64, layers_out=None):
  """Logits [T, vocab] of one sequence; layers_out collects the residual
  stream after every layer."""
  w = {n: t.to(dtype) for n, t in w.items()}
  eps = cfg["norm"]["eps"]
  x = w["embed"][torch.as_tensor(tokens)]
  for i, layer in enumerate(cfg["layers"]):
    p = f"l{i}."
    y = MIXERS[layer["type"]](norm_one_plus(x, w[p + "norm1"], eps), w, p + "mix.", layer["mixer"], eps)
    x = x + norm_one_plus(y, w[p + "norm1b"], eps)
    if layer["mlp"] is not None:
      y = feed_forward(norm_one_plus(x, w[p + "norm2"], eps), w, p + "mlp.")
      x = x + norm_one_plus(y, w[p + "norm2b"], eps)
    if layers_out is not None:
      layers_out.append(x.clone())
  return norm_one_plus(x, w["final.norm"], eps) @ w["head"].T
