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


def sandwich_norm(y, x, w_post, eps):
  return x + _rms(y.float(), eps) * (1.0 + w_post.float())


def add_norm(y, x, mult, w_next, eps):
  x = x + mult * y.float()
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


def chunk_attn(proj, at, H, G, dim, vdim, q_norm, k_norm, sink, mix, scale, eps, chunk, state, rows):
  B, S, _ = proj.shape
  q_at, k_at, v_at = at
  slope = torch.exp2(-8.0 * torch.arange(1, H + 1, device=proj.device, dtype=torch.float32) / H)
  parts = {}
  for b, slot, start, n in _each_row(rows, B, S):
    row = proj[b, :n].float()
    q = (_rms(row[:, q_at:q_at + H * dim].reshape(n, H, dim), eps) * q_norm.float()).to(proj.dtype).float()
    k = (_rms(row[:, k_at:k_at + G * dim].reshape(n, G, dim), eps) * k_norm.float()).to(proj.dtype).float()
    v = row[:, v_at:v_at + G * vdim]
    if mix is not None:
      lam = mix[1].float()
      v = ((1 - lam) * v + lam * mix[0][b, :n].float()).to(proj.dtype).float()
    v = v.reshape(n, G, vdim)
    first, keys, vals = start, k, v
    if state is not None:
      kc, vc = state
      first = start - start % chunk
      keys = torch.cat([kc[slot][:, :start - first].transpose(0, 1).float(), k])
      vals = torch.cat([vc[slot][:, :start - first].transpose(0, 1).float(), v])
    i = torch.arange(start, start + n, device=proj.device)[:, None]
    j = torch.arange(first, start + n, device=proj.device)[None, :]
    s = torch.einsum("nhd,thd->nth", q, keys.repeat_interleave(H // G, dim=1)) * scale
    s = s - (i - j)[:, :, None] * slope
    s = s.masked_fill(((j > i) | (j // chunk != i // chunk))[:, :, None], float("-inf"))
    s0 = sink.float()[None, None]
    p = torch.softmax(torch.cat([s, s0.expand(n, 1, H)], dim=1), dim=1)[:, :-1]
    parts[b] = torch.einsum("nth,the->nhe", p, vals.repeat_interleave(H // G, dim=1)).reshape(n, H * vdim)
    if state is not None:
      last = start + n - 1
      lo = max(start, last - last % chunk)  # what later steps of this chunk read
      kc[slot][:, lo % chunk:last % chunk + 1] = k[lo - start:].transpose(0, 1).to(kc.dtype)
      vc[slot][:, lo % chunk:last % chunk + 1] = v[lo - start:].transpose(0, 1).to(vc.dtype)
  return _scatter(parts, proj, H * vdim)


def _rotate_pairs(x, start, freq):
  """x [n, .., 2 * len(freq)]: neighbours turn by position * freq."""
  pos = torch.arange(start, start + x.shape[0], device=x.device, dtype=torch.float32)
  a = (pos[:, None] * freq.float()).view(x.shape[0], *([1] * (x.dim() - 2)), -1)
  u, v = x[..., 0::2], x[..., 1::2]
  return torch.stack([u * a.cos() - v * a.sin(), v * a.cos() + u * a.sin()], dim=-1).flatten(-2)


def latent_attn(proj, q_at, c_at, H, dim, rot_dim, rank, vdim, norm, up, freq, scale, eps, state, rows, sink=None,
                g_at=None):
  B, S, _ = proj.shape
  parts = {}
  for b, slot, start, n in _each_row(rows, B, S):
    row = proj[b, :n].float()
    q = row[:, q_at:q_at + H * (dim + rot_dim)].reshape(n, H, dim + rot_dim)
    q = torch.cat([q[..., :dim], _rotate_pairs(q[..., dim:], start, freq)], dim=-1)
    c = (_rms(row[:, c_at:c_at + rank], eps) * norm.float()).to(proj.dtype).float()
    t = _rotate_pairs(row[:, c_at + rank:c_at + rank + rot_dim], start, freq).to(proj.dtype).float()
    if state is not None:
      kc, vc = state
      kc[slot, start:start + n] = torch.cat([c, t], dim=-1).to(kc.dtype)
      vc[slot, start:start + n] = c.to(vc.dtype)
      c, t = kc[slot, :start + n].float().split([rank, rot_dim], dim=-1)
    kv = (c @ up.float().t()).to(proj.dtype).float()
    T = c.shape[0]
    k = torch.cat([kv[:, :H * dim].reshape(T, H, dim), t[:, None].expand(T, H, rot_dim)], dim=-1)
    s = torch.einsum("nhd,thd->nth", q, k) * scale
    i = torch.arange(T - n, T, device=proj.device)[:, None]
    s = s.masked_fill((torch.arange(T, device=proj.device)[None] > i)[:, :, None], float("-inf"))
    if sink is not None:
      s = torch.cat([s, sink.float().expand(n, 1, H)], dim=1)
    o = torch.einsum("nth,the->nhe", torch.softmax(s, dim=1)[:, :T], kv[:, H * dim:].reshape(T, H, vdim))
    parts[b] = o.reshape(n, H * vdim)
    if g_at is not None:
      parts[b] = parts[b] * torch.sigmoid(row[:, g_at:g_at + H * vdim])
  return _scatter(parts, proj, H * vdim)


def matrix_memory(proj, at, H, dim, vdim, gate_bias, cap, norm, eps, state, rows):
  B, S, _ = proj.shape
  parts = {}
  for b, slot, start, n in _each_row(rows, B, S):
    q, k, v, g, i, f = (proj[b, :n, a:a + w].float() for a, w in
                        zip(at, (H * dim, H * dim, H * vdim, H * vdim, H, H)))
    q, k, v = (t.reshape(n, H, -1) for t in (q * dim ** -0.5, k, v))
    v = torch.cat([v, torch.ones_like(v[..., :1])], dim=-1)
    i, f = (cap * torch.tanh((t + c.float()) / cap) for t, c in zip((i, f), gate_bias))
    f = F.logsigmoid(f)
    if state is None or start == 0:
      M, m = q.new_zeros(H, vdim + 1, dim), q.new_zeros(H)
    else:
      M, m = state[0][slot][:, :, :dim].clone(), state[1][slot].clone()
    outs = []
    for t in range(n):
      top = torch.maximum(f[t] + m, i[t])
      M = (M * torch.exp(f[t] + m - top)[:, None, None]
           + torch.exp(i[t] - top)[:, None, None] * v[t][:, :, None] * k[t][:, None, :])
      m = top
      o = (M * q[t][:, None, :]).sum(-1)
      outs.append(o[:, :-1] / (torch.maximum(o[:, -1].abs(), torch.exp(-m)) + 1e-6)[:, None])
    o = _rms(torch.stack(outs), eps).reshape(n, H * vdim) * norm.float()
    parts[b] = o * torch.sigmoid(g)
    if state is not None:
      state[0][slot][:, :, :dim] = M
      state[1][slot] = m
  return _scatter(parts, proj, H * vdim)


def embed_pairs(tokens, table, scale, pairs, rule, last, rows):
  B, S = tokens.shape
  row = torch.full_like(tokens, rule["buckets"])
  row[:, 1:] = (tokens[:, :-1] * rule["mul_prev"] + tokens[:, 1:] * rule["mul_cur"]) % rule["buckets"]
  if last is not None:
    for b, slot, start, n in _each_row(rows, B, S):
      if start:
        row[b, 0] = (last[slot, 0].long() * rule["mul_prev"] + tokens[b, 0] * rule["mul_cur"]) % rule["buckets"]
      last[slot, 0] = tokens[b, n - 1]
  return F.embedding(tokens, table).float() * scale + F.embedding(row, pairs).float()


def scalar_norm(x, weight, eps, dtype):
  return (_rms(x.float(), eps) * weight.float()).to(dtype)


def with_conv(h, taps, ring, rows):
  y = short_conv(h, 0, taps, taps.new_zeros(taps.shape[0]), ring, rows, None, False)
  return (h.float() + y.float()).to(h.dtype)


def gated_packed(gu, act):
  g, u = gu.float().chunk(2, dim=-1)
  return (F.gelu(g, approximate="tanh") * u).to(gu.dtype)


def _rotate(x, start, freq, pairs):
  """The first 2 * len(freq) of x's last axis turn by position * freq."""
  n = freq.numel()
  turned, rest = x[..., :2 * n], x[..., 2 * n:]
  if not pairs:
    turned = turned.unflatten(-1, (2, n)).transpose(-1, -2).flatten(-2)
  turned = _rotate_pairs(turned, start, freq)
  if not pairs:
    turned = turned.unflatten(-1, (n, 2)).transpose(-1, -2).flatten(-2)
  return torch.cat([turned, rest], dim=-1)


def _place(p, keep, rows):
  """Row of position p: the first `keep` have their own, the rest a ring."""
  return torch.where(p < keep, p, keep + (p - keep) % max(rows - keep, 1))


def rotary_attn(proj, q_at, source, rule, q_norm, k_norm, freq, lam, state, rows, append):
  r = rule
  B, S, _ = proj.shape
  window = r.window or 1 << 62

  def heads(x, n, norm, start):
    x = x.reshape(x.shape[0], n * r.maps, r.dim)
    if norm is not None:
      x = _rms(x, r.eps) * norm.float()
    x = _rotate(x, start, freq, r.pairs)
    return (_rms(x, r.eps) if r.late_norm else x).to(proj.dtype).float()

  parts = {}
  for b, slot, start, n in _each_row(rows, B, S):
    q = heads(proj[b, :n, q_at:q_at + r.H * r.maps * r.dim].float(), r.H, q_norm, start)
    at = torch.arange(start, start + n, device=proj.device)
    if state is None or append:
      kv, k_at, v_at = source
      k = heads(kv[b, :n, k_at:k_at + r.G * r.maps * r.dim].float(), r.G, k_norm, start)
      v = kv[b, :n, v_at:v_at + r.G * r.vdim].float().view(n, r.G, r.vdim)
    seen = at
    if state is not None:
      kc, vc = state
      R = kc.shape[2]
      first = max(0, start - window + 1)
      seen = torch.cat([torch.arange(0, min(r.keep, first), device=proj.device),
                        torch.arange(first, start + n, device=proj.device)])
      if append:  # of earlier tokens what the cache holds, before newer ones take their rows
        old = _place(seen[:-n], r.keep, R)
        k, v = (torch.cat([c[slot][:, old].transpose(0, 1).float(), t]) for c, t in ((kc, k), (vc, v)))
        stay = (at < r.keep) | (at >= start + n - max(R - r.keep, 1))
        new, row = torch.where(stay)[0], _place(at[stay], r.keep, R)
        kc[slot][:, row] = k[len(old):][new].transpose(0, 1).to(kc.dtype)
        vc[slot][:, row] = v[len(old):][new].transpose(0, 1).to(vc.dtype)
      else:
        here = _place(seen, r.keep, R)
        k, v = (c[slot][:, here].transpose(0, 1).float() for c in (kc, vc))
    dist = at[:, None] - seen[None, :]
    open_ = (dist >= 0) & ((dist < window) | (seen < r.keep)[None])
    per = r.H // r.G
    k = k.unflatten(1, (r.G, r.maps)).repeat_interleave(per, dim=1)
    s = torch.einsum("nhmd,thmd->nthm", q.unflatten(1, (r.H, r.maps)), k) * r.scale
    if r.cap:
      s = r.cap * torch.tanh(s / r.cap)
    p = torch.softmax(s.masked_fill(~open_[:, :, None, None], float("-inf")), dim=1)
    o = torch.einsum("nthm,the->nhme", p, v.repeat_interleave(per, dim=1))
    o = o[:, :, 0] if r.maps == 1 else _rms(o[:, :, 0] - lam * o[:, :, 1], r.eps) * r.gain
    parts[b] = o.reshape(n, r.H * r.vdim)
  return _scatter(parts, proj, r.H * r.vdim)


def gated_unit(proj, y_at, x_at, in_bias, taps, bias, gates, gate_bias, lam, rate, state, rows):
  B, S, _ = proj.shape
  W = lam.numel()
  s, ring = state if state is not None else (None, None)
  u_all = short_conv(proj, x_at, taps, bias, ring, rows, in_bias[1], False)
  parts = {}
  for b, slot, start, n in _each_row(rows, B, S):
    u = u_all[b, :n].float()
    blocks = u.view(n, gates.shape[1], -1)
    r, i = (torch.sigmoid(torch.einsum("nbk,bjk->nbj", blocks, g.float()) + c.float()).reshape(n, W)
            for g, c in zip(gates, gate_bias))
    log_a = -rate * r * F.softplus(lam.float())
    a, x = torch.exp(log_a), torch.sqrt(-torch.expm1(2 * log_a)) * i * u
    M = x.new_zeros(W) if s is None or start == 0 else s[slot].clone()
    outs = []
    for t in range(n):
      M = a[t] * M + x[t]
      outs.append(M)
    y = proj[b, :n, y_at:y_at + W].float() + in_bias[0].float()
    parts[b] = torch.stack(outs) * F.gelu(y, approximate="tanh")
    if s is not None:
      s[slot] = M
  return _scatter(parts, proj, W)


def short_conv(proj, at, taps, bias, ring, rows, in_bias, silu):
  B, S, _ = proj.shape
  C, n_taps = taps.shape
  parts = {}
  for b, slot, start, n in _each_row(rows, B, S):
    x = proj[b, :n, at:at + C]
    if ring is None or start == 0:
      hist = x.new_zeros(n_taps - 1, C, dtype=torch.float32)
    else:
      hist = _history(ring, slot, start, n_taps - 1)
    full = torch.cat([hist, x.float()])
    if in_bias is not None:
      before = min(n_taps - 1, 0 if ring is None else start)  # tokens there are
      full = torch.cat([full[:n_taps - 1 - before], full[n_taps - 1 - before:] + in_bias.float()])
    y = sum(full[j:j + n] * taps[:, j].float() for j in range(n_taps)) + bias.float()
    parts[b] = F.silu(y) if silu else y
    if ring is not None:
      _remember(ring, slot, start, x)
  return _scatter(parts, proj, C)


def selective_scan(x, pre, bc, b_at, c_at, z, z_at, a_log, dt_bias, skip, state, rows):
  B, S, C = x.shape
  n_state = a_log.shape[1]
  A = -torch.exp(a_log.float())
  parts = {}
  for b, slot, start, n in _each_row(rows, B, S):
    xs = x[b, :n].float()
    dt = F.softplus(pre[b, :n].float() + dt_bias.float())
    Bs, Cs = (bc[b, :n, at:at + n_state].float() for at in (b_at, c_at))
    M = xs.new_zeros(C, n_state) if state is None or start == 0 else state[slot].clone()
    outs = []
    for t in range(n):
      M = torch.exp(dt[t][:, None] * A) * M + (dt[t] * xs[t])[:, None] * Bs[t]
      outs.append(M @ Cs[t])
    y = torch.stack(outs) + skip.float() * xs
    parts[b] = y * F.silu(z[b, :n, z_at:z_at + C].float())
    if state is not None:
      state[slot] = M
  return _scatter(parts, x, C)


def expert_mixture(h, router, correction, first, down, ff, rule, act):
  top, groups, keep, scale, softmax, shared, shared_gate, on_input = rule
  D, E = h.shape[-1], router.shape[0] - bool(shared_gate)
  flat = h.reshape(-1, D)
  z = flat.float() @ router.float().t()
  z, open_ = z[:, :E], torch.sigmoid(z[:, E:])
  scores = z if softmax else torch.sigmoid(z)
  choice = scores.detach() if correction is None else scores.detach() + correction.float()
  if keep < groups:
    by_group = choice.view(-1, groups, E // groups)
    score = by_group.topk(min(2, E // groups), dim=-1).values.sum(-1)
    kept = torch.zeros_like(score, dtype=torch.bool).scatter_(1, score.topk(keep, dim=-1).indices, True)
    choice = by_group.masked_fill(~kept[:, :, None], float("-inf")).flatten(1)
  idx = choice.topk(top, dim=-1).indices
  weight = scores.gather(1, idx)
  weight = (torch.softmax(weight, dim=-1) if softmax else weight) * scale
  if shared:
    idx = torch.cat([idx, torch.arange(E, E + shared, device=h.device).expand(len(idx), -1)], dim=1)
    weight = torch.cat([weight, open_.expand(-1, shared) if shared_gate else weight.new_ones(len(idx), shared)], dim=1)
  out = torch.zeros(flat.shape[0], D, dtype=torch.float32, device=h.device)
  for e in range(E + shared):
    tok, k = torch.where(idx == e)
    if tok.numel() == 0:
      continue
    x, F_, w = flat[tok], ff if e < E else first.shape[-2], weight[tok, k, None]
    before, after = (w, 1.0) if on_input else (1.0, w)  # the products are linear in their input
    if act.gated:
      g, u = (F.linear(x, first[e, i, :F_, :D]).float() * before for i in (0, 1))
      g, u = g.clamp(max=act.limit), u.clamp(-act.limit, act.limit)
      a = g * torch.sigmoid(act.alpha * g) * (u + act.plus)
    else:
      a = (F.linear(x, first[e, :F_, :D]).float() * before).relu().square()
    out = out.index_add(0, tok, F.linear(a.to(h.dtype), down[e, :D, :F_]).float() * after)
  return out.to(h.dtype).view(h.shape)
