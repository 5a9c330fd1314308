"""Plain, slow reading of the Tapupel decoder, one function per mechanism.

Float64 on the CPU by default, one sequence at a time, the recurrence stepped
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


def sigmoid(x):
  return 1 / (1 + torch.exp(-x))


def silu(x):
  return x * sigmoid(x)


def softplus(x):
  return torch.log1p(torch.exp(-x.abs())) + x.clamp(min=0)


def gelu_tanh(z):
  return 0.5 * z * (1 + torch.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z ** 3)))


def frequencies(rot):
  """Radians per position of every pair; long wavelengths are slowed down."""
  out = []
  for i in range(rot["dims"] // 2):
    f = rot["base"] ** (-2 * i / rot["dims"])
    s = rot.get("scaling")
    if s is not None:
      wave = 2 * math.pi / f
      if wave > s["original"] / s["low"]:
        f = f / s["factor"]
      elif wave >= s["original"] / s["high"]:
        t = (s["original"] / wave - s["low"]) / (s["high"] - s["low"])
        f = (1 - t) * f / s["factor"] + t * f
    out.append(f)
  return out


def rotate(x, rot, pairs, first=0):
  """x [T,..,n]: the first `dims` of the last axis turn; partners are
  neighbours (pairs) or lie half the turned dims apart."""
  out = x.clone()
  half = rot["dims"] // 2
  at = torch.arange(first, first + x.shape[0], dtype=x.dtype).view(-1, *([1] * (x.dim() - 2)))
  for i, f in enumerate(frequencies(rot)):
    m, n = (2 * i, 2 * i + 1) if pairs else (i, i + half)
    u, v = x[..., m], x[..., n]
    out[..., m] = u * torch.cos(at * f) - v * torch.sin(at * f)
    out[..., n] = v * torch.cos(at * f) + u * torch.sin(at * f)
  return out


def sees(i, j, mask):
  if j > i:
    return False
  return mask is None or i - j < mask["size"] or j < mask["keep_first"]


def attention(q, k, v, scale, mask=None, cap=None):
  """q [T,H,d], k [T,G,d], v [T,G,e]."""
  T, H, _ = q.shape
  per = H // k.shape[1]
  open_ = torch.tensor([[sees(i, j, mask) for j in range(T)] for i in range(T)])
  out = []
  for h in range(H):
    s = q[:, h] @ k[:, h // per].T * scale
    if cap is not None:
      s = cap * torch.tanh(s / cap)
    s = torch.where(open_, s, -torch.inf)
    e = torch.exp(s - s.max(dim=1, keepdim=True).values)
    out.append((e / e.sum(dim=1, keepdim=True)) @ v[:, h // per])
  return torch.stack(out, dim=1)


def window_mixer(h, w, p, m, eps, kept):
  T = h.shape[0]
  H, G, d = m["heads"], m["kv_heads"], m["dim"]
  q, k = (h @ w[p + "q"].T).view(T, H, d), (h @ w[p + "k"].T).view(T, G, d)
  v = k  # as projected
  q, k = (rms(rotate(x, m["rot"], pairs=False), eps) for x in (q, k))
  o = attention(q, k, v, m["scale"], m["mask"], m.get("softcap"))
  return o.reshape(T, -1) @ w[p + "o"].T


def contrast(w, p, diff):
  return (torch.exp((w[p + "lq1"] * w[p + "lk1"]).sum()) - torch.exp((w[p + "lq2"] * w[p + "lk2"]).sum()) + diff)


def difference(q, k, v, scale, lam, diff, eps):
  """q [T,H,2,d], k [T,G,2,d], v [T,G,e]: two attentions over the same values."""
  a1, a2 = (attention(q[:, :, i], k[:, :, i], v, scale) for i in (0, 1))
  return rms(a1 - lam * a2, eps) * (1 - diff)


def differential_mixer(h, w, p, m, eps, kept):
  T = h.shape[0]
  H, G, d, e = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
  q = rotate(rms((h @ w[p + "q"].T).view(T, H, 2, d), eps) * w[p + "q.norm"], m["rot"], pairs=True)
  if m.get("kv_from") is None:
    k = rotate(rms((h @ w[p + "k"].T).view(T, G, 2, d), eps) * w[p + "k.norm"], m["rot"], pairs=True)
    v = (h @ w[p + "v"].T).view(T, G, e)
    kept[p] = k, v
  else:
    k, v = kept[f"l{m['kv_from']}.mix."]
  o = difference(q, k, v, m["scale"], contrast(w, p, m["diff"]), m["diff"], eps)
  return o.reshape(T, -1) @ w[p + "o"].T


def causal_conv(x, taps, bias):
  """x [T,C], taps [C,n]: the last column weighs the current token."""
  n = taps.shape[1]
  padded = torch.cat([x.new_zeros(n - 1, x.shape[1]), x])
  return sum(padded[j:j + x.shape[0]] * taps[:, j] for j in range(n)) + bias


def block_product(u, m, b):
  """u [T, blocks * n], m [blocks, n, n] ([out, in]), b [blocks, n]."""
  parts = u.view(u.shape[0], m.shape[0], -1)
  return torch.cat([parts[:, i] @ m[i].T + b[i] for i in range(m.shape[0])], dim=-1)


def gated_unit(u, ra, ra_b, ri, ri_b, lam):
  """The linear recurrence of real gates: [T, width]."""
  r, i = sigmoid(block_product(u, ra, ra_b)), sigmoid(block_product(u, ri, ri_b))
  log_a = -8 * r * softplus(lam)
  S, out = torch.zeros_like(u[0]), []
  for t in range(u.shape[0]):
    S = torch.exp(log_a[t]) * S + torch.sqrt(-torch.expm1(2 * log_a[t])) * i[t] * u[t]
    out.append(S)
  return torch.stack(out)


def rglru_mixer(h, w, p, m, eps, kept):
  y = gelu_tanh(h @ w[p + "y"].T + w[p + "y.b"])
  u = causal_conv(h @ w[p + "x"].T + w[p + "x.b"], w[p + "conv"], w[p + "conv.b"])
  S = gated_unit(u, w[p + "ra"], w[p + "ra.b"], w[p + "ri"], w[p + "ri.b"], w[p + "lam"])
  return (S * y) @ w[p + "o"].T


def gated_mlp(h, w, p):
  return (silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def route(logits, top):
  """One token: [(expert, weight)]."""
  best = sorted(range(len(logits)), key=lambda e: -logits[e].item())[:top]
  z = torch.exp(logits[best] - logits[best].max())
  return list(zip(best, z / z.sum()))


def expert_mixture(h, w, p, m):
  out = torch.zeros_like(h)
  for t in range(h.shape[0]):
    for e, weight in route(w[p + "router"] @ h[t], m["router"]["top"]):
      out[t] += weight * gated_mlp(h[t], w, f"{p}e{e}.")
  if m.get("shared") is not None:
    out = out + sigmoid(h @ w[p + "shared.sg"].T) * gated_mlp(h, w, p + "shared.")
  return out


def feed_forward(h, w, p, m):
  return gated_mlp(h, w, p) if m["kind"] == "dense" else expert_mixture(h, w, p, m)


MIXERS = {"attention": window_mixer, "attention_2": differential_mixer, "rglru": rglru_mixer}


def forward(tokens, w, cfg, dtype=torch.float64, layers_out=None):
  """Logits [T, vocab] of one sequence; layers_out collects the residual
  stream after every layer."""
  w = {n: t.to(dtype) for n, t in w.items()}
  eps = cfg["norm"]["eps"]
  x = w["embed"][torch.as_tensor(tokens)] * cfg["embedding"]["scale"]
  kept = {}
  for i, layer in enumerate(cfg["layers"]):
    p = f"l{i}."
    y = MIXERS[layer["type"]](x, w, p + "mix.", layer["mixer"], eps, kept)
    x = x + norm_one_plus(y, w[p + "norm1"], eps)
    if layer["mlp"] is not None:
      x = x + norm_one_plus(feed_forward(x, w, p + "mlp.", layer["mlp"]), w[p + "norm2"], eps)
    if layers_out is not None:
      layers_out.append(x.clone())
  return norm_one_plus(x, w["final.norm"], eps) @ w["head"].T
