"""Dispatch of the token mixers' ops and of the fp32-residual norms.

CUDA tensors run the HIP kernels of `_hip_mixers` (hip/mixer_ops.hip) in
bfloat16 or true 32-bit, CPU tensors and training run torch_ref_mixers. A
CUDA tensor never falls back: without the extension the op raises.

A mixer's state is one tuple of tensors per layer whose first dimension is
the slot (engine/kvcache.py, MixerStateCache). `StepRows` says which slot and
which positions a step's rows have, so a step may address any set of slots.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Optional, Tuple

import torch

from xotorch_amd.ops import torch_ref, torch_ref_mixers as ref

_hip = None


def load_hip():
  global _hip
  if _hip is None:
    import importlib
    _hip = importlib.import_module("xotorch_amd.ops._hip_mixers")
  return _hip


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


def row_pad(dim: int) -> int:
  """Key channels of a recurrent state padded to what 16 lanes hold evenly."""
  for per_lane in (1, 2, 3, 4, 6, 8, 12, 16):
    if dim <= 16 * per_lane:
      return 16 * per_lane
  raise ValueError(f"recurrent state with {dim} key channels (at most 256)")


def packed_kv(dtype: torch.dtype, device) -> bool:
  """Whether window-attention caches lie in MFMA fragment order."""
  return dtype == torch.bfloat16 and str(device).startswith("cuda")


# ---------------------------------------------------------------- norms

def prenorm(x, weight, eps: float, dtype: torch.dtype):
  """x fp32 -> RMS norm with a weight around zero, in `dtype`."""
  if _on_hip(x):
    return load_hip().prenorm(x, weight, eps, dtype == torch.bfloat16)
  return ref.prenorm(x, weight, eps, dtype)


def sandwich_norm(y, x, w_post, w_next, eps: float) -> Tuple[torch.Tensor, Optional[torch.Tensor]]:
  """x + norm(y; w_post), and that stream's norm for the next sublayer
  (w_next None: no norm). The stream is fp32; on the HIP path it is updated
  in place."""
  if _on_hip(y):
    return x, load_hip().sandwich_norm(y, x, w_post, w_next, eps)
  return ref.sandwich_norm(y, x, w_post, w_next, eps)


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
    load_hip().window_attn(proj, *at, H, G, dim, vdim, q_norm, k_norm, bucket, rel, scale, eps, window,
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
