"""Torch forms of the token mixers: the CPU path and the training path of
ops/mixer_ops.py (same signatures, plain cache layouts). Everything that the
kernels keep in 32-bit is computed in 32-bit here too. With state None the
functions start from nothing, write nothing and are differentiable.
"""
from __future__ import annotations

import torch
import torch.nn.functional as F


def _rms(x, eps):
  return x * torch.rsqrt(x.pow(2).mean(-1, keepdim=True) + eps)


def prenorm(x, weight, eps, dtype):
  return (_rms(x.float(), eps) * (1.0 + weight.float())).to(dtype)


def sandwich_norm(y, x, w_post, w_next, eps):
  x = x + _rms(y.float(), eps) * (1.0 + w_post.float())
  return x, None if w_next is None else prenorm(x, w_next, eps, y.dtype)


def _each_row(rows, B, S):
  """(row, slot, first position, tokens) of every live row of a step."""
  for b in range(B):
    slot = b if rows.slots is None else int(rows.slots[b])
    if slot < 0:
      continue
    if rows.decode:
      p = rows.positions.reshape(-1)
      yield b, slot, int(p[b] if p.numel() > 1 else p[0]), 1
    else:
      yield b, slot, rows.start, S if rows.lens is None else int(rows.lens[b])


def _scatter(parts, like, width):
  """Rows computed one by one -> [B, S, width], zeros where nothing ran."""
  B, S = like.shape[:2]
  full = []
  for b in range(B):
    part = parts.get(b)
    if part is None:
      part = like.new_zeros(0, width)
    full.append(F.pad(part, (0, 0, 0, S - part.shape[0])))
  return torch.stack(full).to(like.dtype)


def _history(ring, slot, start, count):
  """The last `count` inputs before `start` out of a ring, zeros before 0."""
  M = ring.shape[1]
  out = []
  for p in range(start - count, start):
    out.append(ring[slot, p % M].float() if p >= 0 else torch.zeros_like(ring[slot, 0], dtype=torch.float32))
  return torch.stack(out) if out else ring.new_zeros(0, ring.shape[2], dtype=torch.float32)


def _remember(ring, slot, start, x):
  M = ring.shape[1]
  n = x.shape[0]
  for s in range(max(0, n - M), n):
    ring[slot, (start + s) % M] = x[s].to(ring.dtype)


def window_attn(proj, at, H, G, dim, vdim, q_norm, k_norm, bucket, rel, scale, eps, window, state, rows):
  B, S, _ = proj.shape
  q_at, k_at, v_at, g_at = at
  parts = {}
  for b, slot, start, n in _each_row(rows, B, S):
    row = proj[b, :n].float()
    q = (_rms(row[:, q_at:q_at + H * dim], eps) * q_norm.float()).to(proj.dtype).float().view(n, H, dim)
    k = (_rms(row[:, k_at:k_at + G * dim], eps) * k_norm.float()).to(proj.dtype).float().view(n, G, dim)
    v = row[:, v_at:v_at + G * vdim].view(n, G, vdim)
    first, keys, vals = start, k, v
    if state is not None:
      kc, vc = state
      R = kc.shape[2]
      first = max(0, start - window + 1)
      old = torch.arange(first, start, device=proj.device) % R
      keys = torch.cat([kc[slot][:, old].transpose(0, 1).float(), k])
      vals = torch.cat([vc[slot][:, old].transpose(0, 1).float(), v])
    dist = (torch.arange(start, start + n, device=proj.device)[:, None]
            - torch.arange(first, start + n, device=proj.device)[None, :])
    bias = rel.float()[bucket.long()[dist.clamp(0, bucket.numel() - 1)]]  # [n, keys, H]
    s = torch.einsum("nhd,thd->nth", q, keys.repeat_interleave(H // G, dim=1)) * scale + bias
    s = s.masked_fill(((dist < 0) | (dist >= window))[:, :, None], float("-inf"))
    top = s.amax(1, keepdim=True).clamp(min=0)
    e = torch.exp(s - top)
    p = e / (e.sum(1, keepdim=True) + torch.exp(-top))
    o = torch.einsum("nth,the->nhe", p, vals.repeat_interleave(H // G, dim=1))
    parts[b] = (o * torch.sigmoid(row[:, g_at:g_at + H])[:, :, None]).reshape(n, H * vdim)
    if state is not None:
      keep = min(n, R)
      new = torch.arange(start + n - keep, start + n, device=proj.device) % R
      kc[slot][:, new] = k[n - keep:].transpose(0, 1).to(kc.dtype)
      vc[slot][:, new] = v[n - keep:].transpose(0, 1).to(vc.dtype)
  return _scatter(parts, proj, H * vdim)


def _conv_silu(x, hist, taps):
  n = taps.shape[1]
  full = torch.cat([hist, x])
  y = sum(full[j:j + x.shape[0]] * taps[:, j].float() for j in range(n))
  return F.silu(y)


def _unit(x):
  return x * torch.rsqrt(x.pow(2).sum(-1, keepdim=True) + 1e-6)


def delta_rule(proj, at, H, G, dim, vdim, convs, pre_decay, pre_gate, a_log, dt_bias, norm, eps, state, rows):
  B, S, _ = proj.shape
  taps = convs[0].shape[1]
  widths = (G * dim, G * dim, H * vdim)
  parts = {}
  for b, slot, start, n in _each_row(rows, B, S):
    x = torch.cat([proj[b, :n, a:a + w] for a, w in zip(at, widths)], dim=-1)
    if state is None or start == 0:
      hist = x.new_zeros(taps - 1, x.shape[1], dtype=torch.float32)
      M = x.new_zeros(H, vdim, dim, dtype=torch.float32)
    else:
      hist = _history(state[1], slot, start, taps - 1)
      M = state[0][slot][:, :, :dim].clone()
    q, k, v = _conv_silu(x.float(), hist, torch.cat(convs)).split(widths, dim=-1)
    q = (_unit(q.view(n, G, dim)) * dim ** -0.5).repeat_interleave(H // G, dim=1)
    k = _unit(k.view(n, G, dim)).repeat_interleave(H // G, dim=1)
    v = v.view(n, H, vdim)
    pre = (pre_decay[b, :n].float() + dt_bias.float()).view(n, H, dim)
    g = torch.exp(-torch.exp(a_log.float())[None, :, None] * F.softplus(pre))
    beta = torch.sigmoid(proj[b, :n, at[3]:at[3] + H].float())
    outs = []
    for t in range(n):
      M = M * g[t][:, None, :]
      u = beta[t][:, None] * (v[t] - (M * k[t][:, None, :]).sum(-1))
      M = M + u[:, :, None] * k[t][:, None, :]
      outs.append((M * q[t][:, None, :]).sum(-1))
    o = _rms(torch.stack(outs), eps) * norm.float()
    parts[b] = o.reshape(n, H * vdim) * torch.sigmoid(pre_gate[b, :n].float())
    if state is not None:
      state[0][slot][:, :, :dim] = M
      _remember(state[1], slot, start, x)
  return _scatter(parts, proj, H * vdim)


def token_shift(h, mu, history, rows):
  B, S, D = h.shape
  prev = {}
  for b, slot, start, n in _each_row(rows, B, S):
    x = h[b, :n]
    if history is None or start == 0:
      first = torch.zeros_like(x[:1])
    else:
      first = history[slot, (start - 1) % history.shape[1]][None].to(x.dtype)
    prev[b] = torch.cat([first, x[:-1]])
    if history is not None:
      _remember(history, slot, start, x)
  before = _scatter(prev, h, D).float()
  hf = h.float()
  return torch.stack([(hf + (before - hf) * m.float()).to(h.dtype) for m in mu])


def wkv(r, k, v, gate, pre_decay, w0, u, norm, H, dim, eps, state, rows):
  B, S, _ = r.shape
  parts = {}
  for b, slot, start, n in _each_row(rows, B, S):
    rr, kk, vv = (t[b, :n].float().view(n, H, dim) for t in (r, k, v))
    w = torch.exp(-torch.exp(pre_decay[b, :n].float() + w0.float())).view(n, H, dim)
    bonus = (rr * u.float().view(H, dim) * kk).sum(-1)
    M = rr.new_zeros(H, dim, dim) if state is None or start == 0 else state[slot][:, :, :dim].clone()
    outs = []
    for t in range(n):
      outs.append((M * rr[t][:, None, :]).sum(-1) + bonus[t][:, None] * vv[t])
      M = M * w[t][:, None, :] + vv[t][:, :, None] * kk[t][:, None, :]
    o = _rms(torch.stack(outs), eps).reshape(n, H * dim) * norm.float()
    parts[b] = o * F.silu(gate[b, :n].float())
    if state is not None:
      state[slot][:, :, :dim] = M
  return _scatter(parts, r, H * dim)
