"""Plain, slow reading of the Dupolorn decoder, one function per mechanism.

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


def sigmoid(x):
  return 1 / (1 + torch.exp(-x))


def log_sigmoid(x):
  return x.clamp(max=0) - torch.log1p(torch.exp(-x.abs()))


def gelu_tanh(z):
  return 0.5 * z * (1 + torch.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z ** 3)))


def embed(tokens, w, e):
  """The token's row, scaled, plus a row for the pair it forms with the token
  before it; a sequence's first token has a row of its own, the last."""
  out, b = [], e["bigram"]
  for t, cur in enumerate(tokens):
    row = (tokens[t - 1] * b["mul_prev"] + cur * b["mul_cur"]) % b["buckets"] if t else b["buckets"]
    out.append(w["embed"][cur] * e["scale"] + w["bigram"][row])
  return torch.stack(out)


def with_conv(h, taps):
  """h plus a causal convolution of it; h [T,C], taps [C,n], whose last column
  weighs the current token."""
  n = taps.shape[1]
  padded = torch.cat([h.new_zeros(n - 1, h.shape[1]), h])
  return h + sum(padded[j:j + h.shape[0]] * taps[:, j] for j in range(n))


def depth_average(streams, weights):
  return sum(c * x for c, x in zip(weights, streams, strict=True))


def rotate(x, rot, first=0):
  """x [T,..,n]: neighbours among the first `dims` of the last axis turn."""
  out = x.clone()
  at = torch.arange(first, first + x.shape[0], dtype=x.dtype).view(-1, *([1] * (x.dim() - 2)))
  for i in range(rot["dims"] // 2):
    a = at * rot["base"] ** (-2 * i / rot["dims"])
    u, v = x[..., 2 * i], x[..., 2 * i + 1]
    out[..., 2 * i] = u * torch.cos(a) - v * torch.sin(a)
    out[..., 2 * i + 1] = v * torch.cos(a) + u * torch.sin(a)
  return out


def attention(q, k, v, scale, sink=None):
  """Causal, q and k [T,H,d], v [T,H,e]; a sink per head joins the denominator."""
  T, H, _ = q.shape
  late = torch.ones(T, T, dtype=torch.bool).triu(1)
  out = []
  for h in range(H):
    s = (q[:, h] @ k[:, h].T * scale).masked_fill(late, -torch.inf)
    if sink is not None:
      s = torch.cat([s, sink[h].expand(T, 1)], dim=1)
    e = torch.exp(s - s.max(dim=1, keepdim=True).values)
    out.append((e / e.sum(dim=1, keepdim=True))[:, :T] @ v[:, h])
  return torch.stack(out, dim=1)


def latent_attention(q, c, t, uk, uv, norm, m, eps, sink=None):
  """Queries [T, H * (d + r)], latents [T, R] before their norm, shared key
  parts [T, r] before their turn -> [T, H * e]."""
  T, H, d, r, e = q.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"]
  q = q.reshape(T, H, d + r)
  c = rms(c, eps) * norm
  q = torch.cat([q[..., :d], rotate(q[..., d:], m["rot"])], -1)
  k = torch.cat([(c @ uk.T).view(T, H, d), rotate(t, m["rot"])[:, None].expand(T, H, r)], -1)
  return attention(q, k, (c @ uv.T).view(T, H, e), m["scale"], sink).reshape(T, H * e)


def latent_mixer(h, w, p, m, eps, gated=False):
  R, dkv = m["kv_rank"], h @ w[p + "dkv"].T
  o = latent_attention(h @ w[p + "q"].T, dkv[:, :R], dkv[:, R:], w[p + "uk"], w[p + "uv"], w[p + "dkv.norm"], m, eps,
                       w[p + "sink"] if gated else None)
  if gated:
    o = o * sigmoid(h @ w[p + "g"].T)
  return o @ w[p + "o"].T


def gated_latent_mixer(h, w, p, m, eps):
  return latent_mixer(h, w, p, m, eps, gated=True)


def soft_cap(x, cap):
  return cap * torch.tanh(x / cap)


def matrix_memory(q, k, v, i, f):
  """q, k [T,H,d], v [T,H,e], logs of the input and forget gates [T,H]:
  [T,H,e]. The running maximum starts at 0."""
  T, H, d = q.shape
  S, n, m = q.new_zeros(H, d, v.shape[2]), q.new_zeros(H, d), q.new_zeros(H)
  out = []
  for t in range(T):
    top = torch.maximum(f[t] + m, i[t])
    keep, take = torch.exp(f[t] + m - top), torch.exp(i[t] - top)
    S = keep[:, None, None] * S + take[:, None, None] * k[t][:, :, None] * v[t][:, None, :]
    n = keep[:, None] * n + take[:, None] * k[t]
    m = top
    size = torch.maximum((n * q[t]).sum(-1).abs(), torch.exp(-m)) + 1e-6
    out.append((S * q[t][:, :, None]).sum(1) / size[:, None])
  return torch.stack(out)


def mlstm_mixer(h, w, p, m, eps):
  T, H, d, cap = h.shape[0], m["heads"], m["dim"], m["gate_cap"]
  q, k = (h @ w[p + "q"].T).view(T, H, d) * d ** -0.5, (h @ w[p + "k"].T).view(T, H, d)
  i = soft_cap(h @ w[p + "i"].T + w[p + "i.b"], cap)
  f = log_sigmoid(soft_cap(h @ w[p + "f"].T + w[p + "f.b"], cap))
  o = rms(matrix_memory(q, k, (h @ w[p + "v"].T).view(T, H, m["vdim"]), i, f), eps).reshape(T, -1)
  return (o * w[p + "norm"] * sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


def dense_mlp(h, w, p):
  return (gelu_tanh(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def expert(h, w, p):
  return (h @ w[p + "up"].T).clamp(min=0) ** 2 @ w[p + "down"].T


def route(scores, top):
  return sorted(range(len(scores)), key=lambda e: -scores[e].item())[:top]


def expert_mixture(h, w, p, m):
  """The weight of a chosen expert multiplies its input."""
  out = torch.zeros_like(h)
  for t in range(h.shape[0]):
    s = sigmoid(w[p + "router"] @ h[t])
    for e in route(s, m["router"]["top"]):
      out[t] += expert(s[e] * h[t], w, f"{p}e{e}.")
  if m.get("shared") is not None:
    out = out + expert(h, w, p + "shared.")
  return out


def feed_forward(h, w, p, m):
  return dense_mlp(h, w, p) if m["kind"] == "dense" else expert_mixture(h, w, p, m)


MIXERS = {"latent_attention": latent_mixer, "latent_attention_2": gated_latent_mixer, "mlstm": mlstm_mixer}


def forward(tokens, w, cfg, dtype=torch.float64, layers_out=None):
  """Logits [T, vocab] of one sequence; layers_out collects the stream that
  every layer hands on."""
  w = {n: t.to(dtype) for n, t in w.items()}
  eps = cfg["norm"]["eps"]
  x = embed(tokens, w, cfg["embedding"])
  streams = [x]
  for i, layer in enumerate(cfg["layers"]):
    p = f"l{i}."
    h = with_conv(rms(x, eps) * w[p + "norm1"], w[p + "canon1"])
    x_new = x + MIXERS[layer["type"]](h, w, p + "mix.", layer["mixer"], eps)
    if layer["mlp"] is not None:
      x_new = x_new + feed_forward(rms(x, eps) * w[p + "norm2"], w, p + "mlp.", layer["mlp"])
    streams.append(x_new)
    x = depth_average(streams, w[p + "dwa"])
    if layers_out is not None:
      layers_out.append(x.clone())
  return soft_cap((rms(x, eps) * w["final.norm"]) @ w["head"].T, cfg["logit_softcap"])
