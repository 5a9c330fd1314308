"""Dispatch of the token mixers' ops and of the fp32-residual norms.

CUDA tensors run the HIP kernels of `_hip_mixers`, `_hip_attn`, `_hip_latent`,
`_hip_scan`, `_hip_rotary`, `_hip_lru`, `_hip_mlstm`, `_hip_stream` and
`_hip_experts` (hip/*.hip) in bfloat16 or true 32-bit, CPU tensors and training run torch_ref_mixers. A CUDA
tensor never falls back: without the extension the op raises.

A mixer's state is one tuple of tensors per layer whose first dimension is
the slot (engine/kvcache.py, MixerStateCache). `StepRows` says which slot and
which positions a step's rows have, so a step may address any set of slots.
"""
from __future__ import annotations

from dataclasses import dataclass, field
from typing import Dict, NamedTuple, Optional, Tuple, Union

import torch

from xotorch_amd.ops import torch_ref, torch_ref_mixers as ref

_hip = {}


def load_hip(name: str = "_hip_mixers"):
  if name not in _hip:
    import importlib
    _hip[name] = importlib.import_module(f"xotorch_amd.ops.{name}")
  return _hip[name]


def _on_hip(t: torch.Tensor) -> bool:
  """HIP path for CUDA tensors outside of training (the kernels have no
  backward; the torch functions are differentiable)."""
  return t.is_cuda and not (torch.is_grad_enabled() and t.requires_grad)


@dataclass
class StepRows:
  """Rows of one step. A prefill chunk starts at position `start` in every
  row and brings lens[b] tokens (None: all of the chunk; the rest is padding).
  A decode step brings one token per row at positions[b] (or positions[0] for
  all). Row b lives in state slot slots[b] (None: b); slot -1 is a parked
  row, which neither reads nor writes any state."""
  decode: bool
  start: int = 0
  positions: Optional[torch.Tensor] = None
  slots: Optional[torch.Tensor] = None
  lens: Optional[torch.Tensor] = None
  # what of a layer [B, S, *] later layers and ring stages read, by name
  carried: Dict[str, torch.Tensor] = field(default_factory=dict)
  # (state, source, key norm) of layers whose keys and values others read
  kept: Dict[int, tuple] = field(default_factory=dict)
  streamed: bool = False  # whether the stream between layers is read by others than layers
  # the stream as it was after the embedding and after every layer so far
  depth: Optional["Depth"] = None


def row_pad(dim: int) -> int:
  """Key channels of a recurrent state padded to what 16 lanes hold evenly."""
  for per_lane in (1, 2, 3, 4, 6, 8, 12, 16):
    if dim <= 16 * per_lane:
      return 16 * per_lane
  raise ValueError(f"recurrent state with {dim} key channels (at most 256)")


def packed_kv(dtype: torch.dtype, device) -> bool:
  """Whether window-attention caches lie in MFMA fragment order."""
  return dtype == torch.bfloat16 and str(device).startswith("cuda")


_side: Dict[int, "torch.cuda.Stream"] = {}


def side_by_side(first, second):
  """Results of two functions that do not depend on each other. In a captured step
  they are branches of the graph, so that what is bound by latency overlaps.
  Whatever the second allocates is used up before the current stream forks again."""
  if not (torch.cuda.is_available() and torch.cuda.is_current_stream_capturing()):
    return first(), second()
  main = torch.cuda.current_stream()
  side = _side.setdefault(main.device_index, torch.cuda.Stream(main.device_index))
  side.wait_stream(main)
  with torch.cuda.stream(side):
    b = second()
  a = first()
  main.wait_stream(side)
  return a, b


# ---------------------------------------------------------------- norms

class _Stream:
  """In the place of a norm's weight: the stream is read as it is."""


STREAM = _Stream()


def prenorm(x, weight, eps: float, dtype: torch.dtype):
  """x fp32 -> RMS norm with a weight around zero (STREAM: x itself), in
  `dtype`."""
  if weight is STREAM:
    return x.to(dtype)
  if _on_hip(x):
    return load_hip().prenorm(x, weight, eps, dtype == torch.bfloat16)
  return ref.prenorm(x, weight, eps, dtype)


class Weighted(NamedTuple):
  """sum_k weight[t, k] y[row[t, k]] for every token t, not yet summed."""
  y: torch.Tensor
  row: torch.Tensor
  weight: Optional[torch.Tensor]  # None: all one


def sandwich_norm(y: Union[torch.Tensor, Weighted], x, w_post, w_next,
                  eps: float) -> Tuple[torch.Tensor, Optional[torch.Tensor]]:
  """x + norm(y; w_post), and that stream's norm for the next sublayer
  (w_next None: no norm; STREAM: the stream as it is). The stream is fp32; on
  the HIP path it is updated in place."""
  copy = w_next is STREAM
  if isinstance(y, Weighted):
    return x, load_hip().sandwich_norm(y.y, x, w_post, None if copy else w_next, eps, copy, y.row, y.weight)
  if _on_hip(y):
    return x, load_hip().sandwich_norm(y, x, w_post, None if copy else w_next, eps, copy)
  x = ref.sandwich_norm(y, x, w_post, eps)
  return x, None if w_next is None else prenorm(x, w_next, eps, y.dtype)


def add_norm(y: Union[torch.Tensor, Weighted], x, mult: float, w_next, eps: float):
  """x + mult * y, and that stream's norm for the next sublayer (w_next None:
  no norm). The stream is fp32; on the HIP path it is updated in place."""
  if isinstance(y, Weighted):
    return x, load_hip("_hip_experts").add_norm(y.y, y.row, y.weight, x, w_next, mult, eps)
  if _on_hip(y):
    return x, load_hip("_hip_experts").add_norm(y, None, None, x, w_next, mult, eps)
  return ref.add_norm(y, x, mult, w_next, eps)


# ------------------------------------- embedding of pairs, averages over depth

class Depth:
  """The streams that averages over depth read: `streams[j]` in fp32, as views of
  one slab on the HIP path, whose kernels fill it. before: weights of the last
  average, where that itself was not written."""

  def __init__(self, like, tokens: tuple, count: int, width: Optional[int] = None, keep: bool = True):
    self.slab = self.before = None
    self.keep = keep  # whether averages between layers are read by others
    if _on_hip(like):
      self.slab = torch.empty(count, *tokens, width or like.shape[-1], dtype=torch.float32, device=like.device)
    self.streams = []

  def place(self):
    """The slab's next place, which counts as filled."""
    self.streams.append(self.slab[len(self.streams)])
    return self.streams[-1]

  def add(self, x):
    if self.slab is not None:
      self.place().copy_(x)
    else:
      self.streams.append(x)


class Reads(NamedTuple):
  """What a layer reads of the stream: RMS norms with one number each, and a
  causal convolution over time that is added to the first."""
  norms: Tuple[torch.Tensor, ...]
  taps: Optional[torch.Tensor] = None
  ring: Optional[torch.Tensor] = None  # the convolution's last inputs


def embed_pairs(tokens, table, scale: float, pairs, rule: dict, last, rows: StepRows):
  """fp32 rows of `table` times scale plus rows (previous token * mul_prev + token
  * mul_cur) mod buckets of `pairs`; row `buckets` for a sequence's first token.
  last: int32 [slots, 1], the token before a row's step, updated. The result is
  the first of rows.depth."""
  if _on_hip(table):
    x = rows.depth.place()
    load_hip("_hip_stream").embed_pairs(tokens, table, scale, pairs, rule["buckets"], rule["mul_prev"], rule["mul_cur"],
                                        last, rows.slots, rows.positions, rows.lens, rows.start, rows.decode, x)
    return x
  x = ref.embed_pairs(tokens, table, scale, pairs, rule, last, rows)
  rows.depth.add(x)
  return x


def input_conv(h, taps, ring, rows: StepRows):
  """h plus its causal convolution over time."""
  if _on_hip(h):
    return load_hip("_hip_scan").short_conv(h, 0, taps, None, None, False, ring, rows.slots, rows.positions, rows.lens,
                                            rows.start, rows.decode, True)
  return ref.with_conv(h, taps, ring, rows)


def read_stream(x, reads: Reads, eps: float, dtype: torch.dtype, rows: StepRows):
  """A tuple: what `reads` says of the fp32 stream, in `dtype`."""
  if _on_hip(x):
    return _depth_norm(None, None, x, None, None, reads, eps, dtype, rows)[1]
  h = [ref.scalar_norm(x, g, eps, dtype) for g in reads.norms]
  if reads.taps is not None:
    h[0] = input_conv(h[0], reads.taps, reads.ring, rows)
  return tuple(h)


def depth_norm(y, z, x, weights, reads: Optional[Reads], eps: float, dtype: torch.dtype, rows: StepRows):
  """One layer's end: x + y + z joins rows.depth, the sum of its streams times
  `weights` is the new stream. Returns it and what is read of it next. On the HIP
  path a stream between two layers is None, unless it is asked for: the next
  layer's end makes it again of what it reads anyway."""
  if _on_hip(y):
    return _depth_norm(y, z, x, rows.depth, weights, reads, eps, dtype, rows)
  new = x + y.float() if z is None else x + y.float() + z.float()
  rows.depth.add(new)
  x = sum(c * t for c, t in zip(weights.float(), rows.depth.streams, strict=True))
  return x, None if reads is None else read_stream(x, reads, eps, dtype, rows)


def _depth_norm(y, z, x, depth, weights, reads, eps, dtype, rows):
  take = weigh = None
  if isinstance(z, Weighted):
    z, take, weigh = z
  norms, taps, ring = reads if reads is not None else ((), None, None)
  fused = rows.decode and taps is not None  # one token a row: the convolution's other inputs are in its state
  done = len(depth.streams) if depth is not None else 0
  slab, before, keep = (depth.slab, depth.before, depth.keep or taps is None) if depth is not None else (None, None, False)
  x, *h = load_hip("_hip_stream").depth_norm(
    y, z, take, weigh, x, None if x is not None else before, slab, done, weights, keep, norms[0] if norms else None,
    norms[1] if len(norms) > 1 else None, taps if fused else None, ring if fused else None, rows.slots, rows.positions,
    eps, dtype == torch.bfloat16)
  if depth is not None:
    depth.place()
    depth.before = weights
  h = h[:len(norms)]
  if taps is not None and not fused:
    h[0] = input_conv(h[0], taps, ring, rows)
  return x, tuple(h)


def soft_cap(x, cap: float):
  """cap * tanh(x / cap) in fp32."""
  if _on_hip(x):
    return load_hip("_hip_stream").soft_cap(x, cap)
  return cap * torch.tanh(x.float() / cap)


def gated_packed(gu, act: str):
  """gelu_tanh(gate) * up on a packed [.., 2I] projection of any width and dtype."""
  if act != "gelu_tanh":
    raise ValueError(f"unknown activation {act!r}")
  if _on_hip(gu):
    return load_hip("_hip_stream").geglu_packed(gu)
  return ref.gated_packed(gu, act)


def swiglu_packed(gu):
  """silu(gate) * up on a packed [.., 2I] projection of any width and dtype."""
  if _on_hip(gu):
    return load_hip().swiglu_packed(gu)
  return torch_ref.swiglu_packed(gu)


# ---------------------------------------------------------------- mixers

def _out(out, like, width):
  return out if out is not None else torch.empty(*like.shape[:-1], width, dtype=like.dtype, device=like.device)


def window_attn(proj, at, H: int, G: int, dim: int, vdim: int, q_norm, k_norm, bucket, rel,
                scale: float, eps: float, window: int, state, rows: StepRows,
                out=None, out_at: int = 0, out_scale: float = 1.0):
  """Sliding-window attention with RMS norms over the whole q and k
  projections, a learned bias per distance, a zero-score sink in the softmax
  and one sigmoid gate per head. `at` gives the columns of q, k, v and gate in
  `proj`; the result lands in columns out_at.. of `out`."""
  if _on_hip(proj):
    out = _out(out, proj, H * vdim)
    load_hip("_hip_attn").window_attn(proj, *at, H, G, dim, vdim, q_norm, k_norm, bucket, rel, scale, eps, window,
                           state[0], state[1], rows.slots, rows.positions, rows.lens, rows.start,
                           rows.decode, out, out_at, out_scale)
    return out
  return ref.window_attn(proj, at, H, G, dim, vdim, q_norm, k_norm, bucket, rel, scale, eps, window,
                         state, rows) * out_scale


def delta_rule(proj, at, H: int, G: int, dim: int, vdim: int, convs, pre_decay, pre_gate,
               a_log, dt_bias, norm, eps: float, state, rows: StepRows,
               out=None, out_at: int = 0, out_scale: float = 1.0):
  """Gated delta rule with short causal convolutions, unit q and k, a decay
  per key channel, and a gated RMS norm per head. `at` gives the columns of
  q, k, v and beta in `proj`; convs are the taps of q, k, v; pre_decay and
  pre_gate are the low-rank projections before softplus and sigmoid."""
  if _on_hip(proj):
    out = _out(out, proj, H * vdim)
    load_hip().delta_rule(proj, *at, H, G, dim, vdim, *convs, pre_decay, pre_gate, a_log, dt_bias, norm, eps,
                          state[0], state[1], rows.slots, rows.positions, rows.lens, rows.start,
                          rows.decode, out, out_at, out_scale)
    return out
  return ref.delta_rule(proj, at, H, G, dim, vdim, convs, pre_decay, pre_gate, a_log, dt_bias, norm, eps,
                        state, rows) * out_scale


def token_shift(h, mu, history, rows: StepRows):
  """h + (previous token's h - h) * mu for every row of mu: [n, B, S, D]."""
  if _on_hip(h):
    return load_hip().token_shift(h, mu, history, rows.slots, rows.positions, rows.lens, rows.start, rows.decode)
  return ref.token_shift(h, mu, history, rows)


def tanh(x):
  if _on_hip(x):
    return load_hip().tanh(x)
  return torch.tanh(x.float()).to(x.dtype)


def wkv(r, k, v, gate, pre_decay, w0, u, norm, H: int, dim: int, eps: float, S, rows: StepRows):
  """Decayed outer-product memory with a bonus for the current token, an RMS
  norm per head, a weight and a silu gate. Inputs [B, S, H*dim]."""
  if _on_hip(r):
    return load_hip().wkv(r, k, v, gate, pre_decay, w0, u, norm, H, dim, eps, S,
                          rows.slots, rows.positions, rows.lens, rows.start, rows.decode)
  return ref.wkv(r, k, v, gate, pre_decay, w0, u, norm, H, dim, eps, S, rows)


def chunk_attn(proj, at, H: int, G: int, dim: int, vdim: int, q_norm, k_norm, sink, mix, scale: float, eps: float,
               chunk: int, state, rows: StepRows, out=None, out_at: int = 0, out_scale: float = 1.0):
  """Attention within chunks of the sequence: RMS norms per head, scores minus
  2^(-8 (h+1) / H) times the distance, a learned sink per head. `mix`: (values
  of an earlier layer, how much of them) or None. `at` gives the columns of q,
  k and v in `proj`."""
  if _on_hip(proj):
    out = _out(out, proj, H * vdim)
    load_hip("_hip_attn").chunk_attn(proj, *at, H, G, dim, vdim, q_norm, k_norm, sink, *(mix or (None, None)), scale,
                                     eps, chunk, state[0], state[1], rows.slots, rows.positions, rows.lens, rows.start,
                                     rows.decode, out, out_at, out_scale)
    return out
  return ref.chunk_attn(proj, at, H, G, dim, vdim, q_norm, k_norm, sink, mix, scale, eps, chunk, state,
                        rows) * out_scale


def latent_attn(proj, q_at: int, c_at: int, H: int, dim: int, rot_dim: int, rank: int, vdim: int, norm, up, freq,
                scale: float, eps: float, state, rows: StepRows, sink=None, g_at: Optional[int] = None, out=None,
                out_at: int = 0, out_scale: float = 1.0):
  """Causal attention over normed latents (`rank` columns of proj from c_at on,
  then a rotated key part that all heads share). `up` expands a latent into the
  keys, then the values of all heads. sink: a score per head that joins the
  denominator; g_at: columns whose sigmoid multiplies the result. Prompts expand
  the latents of all earlier tokens; decode steps fold the expansion into query
  and output."""
  if not _on_hip(proj):
    return ref.latent_attn(proj, q_at, c_at, H, dim, rot_dim, rank, vdim, norm, up.weight, freq, scale, eps, state,
                           rows, sink, g_at) * out_scale
  hip = load_hip("_hip_latent")
  out = _out(out, proj, H * vdim)
  sizes = (q_at, c_at, H, dim, rot_dim, rank, norm, freq, eps, state[0], state[1], rows.slots)
  if rows.decode:
    qn, qr = hip.latent_append_step(proj, *sizes, rows.positions)
    w = up.weight
    folded = torch.bmm(qn, w[:H * dim].view(H, dim, rank))
    seen = hip.latent_decode(folded, qr, state[0], state[1], scale, rows.slots, rows.positions, sink)
    o = torch.bmm(seen, _value_weights(up, H, dim))  # [H, B, vdim]
    hip.gather_heads(o, proj if g_at is not None else None, g_at or 0, out, out_at, out_scale)
    return out
  q, latents, turned = hip.latent_append(proj, *sizes, rows.lens, rows.start)
  k, v, n = hip.pack_heads(up(latents), turned, H, dim, rot_dim, vdim)
  load_hip("_hip_attn").causal_attn(q, k, v, dim + rot_dim, vdim, n, scale, rows.slots, rows.lens, rows.start, out,
                                    out_at, out_scale, sink, proj if g_at is not None else None, g_at or 0)
  return out


def matrix_memory(proj, at, H: int, dim: int, vdim: int, gate_bias, cap: float, norm, eps: float, state, rows: StepRows,
                  out=None, out_at: int = 0, out_scale: float = 1.0):
  """S = e^f S + e^i k v^T, read with q and divided by max(|n q|, 1), n the same
  sum of the keys alone; all relative to a running maximum of the exponents (from
  0 on), which a small constant in the divisor sees. An RMS norm per head, `norm`
  and a sigmoid gate follow. `at` gives the columns of q, k, v, the output gate
  and the logs of input and forget gate before cap, bias and sigmoid."""
  if not _on_hip(proj):
    return ref.matrix_memory(proj, at, H, dim, vdim, gate_bias, cap, norm, eps, state, rows) * out_scale
  out = _out(out, proj, H * vdim)
  load_hip("_hip_mlstm").matrix_memory(proj, *at, H, dim, vdim, gate_bias, cap, norm, eps, state[0], state[1], rows.slots,
                                       rows.positions, rows.lens, rows.start, rows.decode, out, out_at, out_scale)
  return out


def _value_weights(up, H: int, dim: int):
  """The value half of `up` as [H, rank, vdim], kept with the module."""
  w = up.weight
  key = (w.data_ptr(), w._version)
  if getattr(up, "_values_key", None) != key:
    up._values = w[H * dim:].detach().view(H, -1, w.shape[1]).transpose(1, 2).contiguous()
    up._values_key = key
  return up._values


class AttnRule(NamedTuple):
  """Sizes and constants of rotary attention (models.mixers.RotaryAttention)."""
  H: int
  G: int
  dim: int
  vdim: int
  maps: int          # 2: differential
  scale: float
  cap: float         # 0: scores are not capped
  window: int        # 0: causal
  keep: int          # first tokens that stay in sight of the window
  pairs: bool        # neighbours turn together
  late_norm: bool    # a norm without a weight after the rotation
  eps: float
  gain: float        # of the normed difference of the maps


def rotary_attn(proj, q_at: int, source, rule: AttnRule, q_norm, k_norm, freq, lam, state, rows: StepRows, append: bool,
                out=None, out_at: int = 0, out_scale: float = 1.0):
  """Attention with rotary positions over `state`'s keys and values. source:
  (tensor, column of the keys, column of the values), appended to the state
  first, unless another layer has done so (`append` False). freq: radians per
  position of each pair. lam: what the second map is weighed with."""
  if not _on_hip(proj):
    return ref.rotary_attn(proj, q_at, source, rule, q_norm, k_norm, freq, lam, state, rows, append) * out_scale
  out = _out(out, proj, rule.H * rule.vdim)
  kv, k_at, v_at = source if append else (None, 0, 0)
  load_hip("_hip_rotary").rotary_attn(proj, q_at, kv, k_at, v_at, *rule, q_norm, k_norm, freq, lam, state[0], state[1],
                                      rows.slots, rows.positions, rows.lens, rows.start, rows.decode, out, out_at,
                                      out_scale)
  return out


def short_conv(proj, at: int, taps, bias, ring, rows: StepRows, in_bias=None, silu: bool = False):
  """Causal convolution per channel over the columns of `proj` from `at` on
  (plus `in_bias`; zeros come before the first token), and silu: [B, S,
  channels]."""
  if _on_hip(proj):
    return load_hip("_hip_scan").short_conv(proj, at, taps, bias, in_bias, silu, ring, rows.slots, rows.positions,
                                            rows.lens, rows.start, rows.decode)
  return ref.short_conv(proj, at, taps, bias, ring, rows, in_bias, silu)


def conv_silu(proj, at: int, taps, bias, ring, rows: StepRows):
  return short_conv(proj, at, taps, bias, ring, rows, silu=True)


def gated_unit(proj, y_at: int, x_at: int, in_bias, taps, bias, gates, gate_bias, lam, rate: float, state,
               rows: StepRows, out=None, out_at: int = 0, out_scale: float = 1.0):
  """S = a S + sqrt(1 - a^2) i u per channel, times gelu(y). u: the convolution
  of the columns from x_at on; y: those from y_at on; both with a row of
  in_bias [2, W] (y, x). Gates r and i: sigmoid of block-diagonal products of u
  (gates [2, blocks, n, n], gate_bias [2, blocks, n]); log a = -rate r
  softplus(lam)."""
  if not _on_hip(proj):
    return ref.gated_unit(proj, y_at, x_at, in_bias, taps, bias, gates, gate_bias, lam, rate, state, rows) * out_scale
  hip = load_hip("_hip_lru")
  out = _out(out, proj, lam.numel())
  if rows.decode:
    hip.gated_unit_step(proj, y_at, x_at, in_bias, taps, bias, gates, gate_bias, lam, rate, state[0], state[1],
                        rows.slots, rows.positions, out, out_at, out_scale)
    return out
  u = short_conv(proj, x_at, taps, bias, state[1], rows, in_bias[1])
  hip.gated_unit(u, proj, y_at, in_bias, gates, gate_bias, lam, rate, state[0], rows.slots, rows.lens, rows.start, out,
                 out_at, out_scale)
  return out


def selective_scan(x, pre, bc, b_at: int, c_at: int, z, z_at: int, a_log, dt_bias, skip, state, rows: StepRows,
                   out=None, out_at: int = 0, out_scale: float = 1.0):
  """Selective state space scan of x [B, S, C] with step sizes softplus(pre +
  dt_bias), decays exp(-step exp(a_log)), B and C in columns of `bc`, a skip
  and a silu gate in columns of `z`."""
  if _on_hip(x):
    out = _out(out, x, x.shape[-1])
    load_hip("_hip_scan").selective_scan(x, pre, bc, b_at, c_at, z, z_at, a_log, dt_bias, skip, state, rows.slots,
                                         rows.positions, rows.lens, rows.start, rows.decode, out, out_at, out_scale)
    return out
  return ref.selective_scan(x, pre, bc, b_at, c_at, z, z_at, a_log, dt_bias, skip, state, rows) * out_scale


# ---------------------------------------------------------------- experts

class Routing(NamedTuple):
  """How tokens choose experts and weigh them (models.experts)."""
  top: int
  groups: int
  keep: int               # groups that stay open
  scale: float
  softmax: bool = False   # weights are the softmax over the chosen logits
  shared: int = 0         # experts after the routed ones that every token uses
  shared_gate: bool = True  # their weight is the sigmoid of the router's last row (else one)
  on_input: bool = False  # weights multiply the experts' input, not their output


class GatedAct(NamedTuple):
  """min(g, limit) sigmoid(alpha min(g, limit)) (clamp(u, +-limit) + plus)."""
  alpha: float
  limit: float
  plus: float
  gated: bool = True


class _Relu2:
  gated = False


RELU2 = _Relu2()


def expert_mixture(h, router, correction, first, down, ff: int, rule: Routing, act):
  """Weighted sum of each token's best experts and of the shared ones. first
  [E, 2, F, K] (gate and up of a gated activation) or [E, F, K] and down [E, D, F]
  are padded with zeros past the model's width and `ff`."""
  if _on_hip(h):
    hip = load_hip("_hip_experts")
    flat = h.view(-1, h.shape[-1])
    # weights are per token and choice, for the sum, or per row, for the first product
    weight, row, *places = hip.route(flat, router, correction, *rule)
    alpha, limit, plus = act[:3] if act.gated else (0.0, 0.0, 0.0)
    g = hip.expert_product(flat, first, *places, hip.GATED if act.gated else hip.RELU2, alpha, limit, plus,
                           weight if rule.on_input else None)
    return Weighted(hip.expert_product(g, down, *places, hip.PLAIN), row, None if rule.on_input else weight)
  return ref.expert_mixture(h, router, correction, first, down, ff, rule, act)
