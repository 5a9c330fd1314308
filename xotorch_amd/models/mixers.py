"""Token mixers beyond plain GQA attention, composable per layer.

A design that lists its layers (ModelConfig.layer_specs) names a mixer for
each; MIXERS maps that name to a class here. Every constant of a mechanism is
a parameter of its branch, so another design can use it with its own.

Branches that read projections of the layer's input (the attentions,
`GatedDeltaRule`, `SelectiveScan`, `GatedLinearUnit`, `MatrixMemory`) are combined by `BranchMixer`: ONE fused input GEMM over
the parts of all branches and ONE output GEMM over their concatenated
activations (branch weights fold into the activations in fp32), however many
branches run side by side. `WKVMixer` shifts its input per projection and so
keeps GEMMs of its own.

State lives outside (engine/kvcache.py): each class says in `state_spec` what
one slot holds and gets the tensors back in `forward`.
"""
from __future__ import annotations

import math
from typing import Dict, List, Optional, Tuple

import torch
import torch.nn as nn

from xotorch_amd.models.llama import XotLinear
from xotorch_amd.ops import mixer_ops as mo

StateSpec = Dict[str, Tuple[tuple, torch.dtype]]  # name -> (shape per slot, dtype)


def _up(n: int, to: int) -> int:
  return -(-n // to) * to


def distance_buckets(rows: int, far: int, length: int) -> torch.Tensor:
  """Bucket of every distance 0..length-1: the first half of `rows` one each,
  the rest logarithmic up to distance `far`, clamped to the last."""
  half = rows // 2
  out = []
  for n in range(length):
    if n < half:
      out.append(n)
      continue
    # the nudge keeps exact powers on their own side of the floor
    steps = math.log(n / half) / math.log(far / half) * (rows - half)
    out.append(min(rows - 1, half + math.floor(steps + 1e-9)))
  return torch.tensor(out, dtype=torch.int32)


class WindowBiasAttention(nn.Module):
  """GQA attention over a sliding window: RMS norm over the whole q and k
  projections, no rotation, a learned bias per distance bucket, a sink of
  score zero in the softmax, one sigmoid output gate per head."""

  hip = ("_hip_attn",)

  def __init__(self, dim: int, p: dict, eps: float):
    super().__init__()
    self.H, self.G, self.dim, self.vdim = p["heads"], p["kv_heads"], p["dim"], p["vdim"]
    if self.H % self.G:
      raise ValueError(f"{self.H} query heads do not divide into {self.G} key/value heads")
    self.scale, self.window, self.far, self.eps = float(p["scale"]), int(p["mask"]["size"]), p["bias_max"], eps
    if self.window < 1:
      raise ValueError(f"window of {self.window} tokens")
    self.parts = [("q", self.H * self.dim), ("k", self.G * self.dim), ("v", self.G * self.vdim), ("g", self.H)]
    self.width = self.H * self.vdim
    self.q_norm = nn.Parameter(torch.ones(self.H * self.dim))
    self.k_norm = nn.Parameter(torch.ones(self.G * self.dim))
    self.rel = nn.Parameter(torch.zeros(p["buckets"], self.H))
    self.init_ranges = {"q_norm": (0.8, 1.2), "k_norm": (0.8, 1.2), "rel": (-0.5, 0.5)}
    self.register_buffer("bucket", torch.empty(0, dtype=torch.int32), persistent=False)
    self.reset_tables()

  def reset_tables(self, device=None):
    # the last bucket starts at distance `far` at the latest, so the table
    # ends there and longer distances read its last entry
    length = min(self.window, max(int(math.ceil(self.far)), self.rel.shape[0] // 2) + 1)
    self.bucket = distance_buckets(self.rel.shape[0], self.far, length).to(device or self.bucket.device)

  @staticmethod
  def state_spec(p: dict, capacity: int, dtype: torch.dtype, device) -> StateSpec:
    G, d, e = p["kv_heads"], p["dim"], p["vdim"]
    ring = min(p["mask"]["size"], capacity)  # only a window of keys is ever read
    if mo.packed_kv(dtype, device):
      ring = _up(ring, 32)
      # MFMA fragment order, dims padded with zeros: 16-token x 32-dim key
      # tiles, 32-token x 16-dim value tiles
      return {"k": ((G, ring // 16, _up(d, 32) // 32, 64, 8), dtype),
              "v": ((G, _up(e, 16) // 16, ring // 32, 64, 8), dtype)}
    return {"k": ((G, ring, d), dtype), "v": ((G, ring, e), dtype)}

  @staticmethod
  def param_count(dim: int, p: dict) -> int:
    H, G, d, e = p["heads"], p["kv_heads"], p["dim"], p["vdim"]
    return dim * (H * d + G * d + G * e + H + H * e) + H * d + G * d + p["buckets"] * H

  def forward(self, h, proj, at, state, rows, **out):
    return mo.window_attn(proj, [at[n] for n, _ in self.parts], self.H, self.G, self.dim, self.vdim,
                          self.q_norm, self.k_norm, self.bucket, self.rel, self.scale, self.eps, self.window,
                          state, rows, **out)


class GatedDeltaRule(nn.Module):
  """Gated delta rule: short causal convolutions on q, k, v, unit q and k, a
  decay per head and key channel and an output gate through low-rank pairs,
  fp32 state [heads, vdim, dim]."""

  def __init__(self, dim: int, p: dict, eps: float):
    super().__init__()
    self.H, self.G, self.dim, self.vdim = p["heads"], p["kv_heads"], p["dim"], p["vdim"]
    if self.H % self.G:
      raise ValueError(f"{self.H} heads do not divide into {self.G} key heads")
    self.eps = eps
    H, G, d, e, taps = self.H, self.G, self.dim, self.vdim, p["conv"]
    self.ranks = (p["decay_rank"], p["gate_rank"])
    self.parts = [("q", G * d), ("k", G * d), ("v", H * e), ("a1", self.ranks[0]), ("g1", self.ranks[1]), ("b", H)]
    self.width = H * e
    self.q_conv = nn.Parameter(torch.zeros(G * d, taps))
    self.k_conv = nn.Parameter(torch.zeros(G * d, taps))
    self.v_conv = nn.Parameter(torch.zeros(H * e, taps))
    self.decay_up = XotLinear(self.ranks[0], H * d, bias=False)
    self.gate_up = XotLinear(self.ranks[1], H * e, bias=False)
    self.a_log = nn.Parameter(torch.zeros(H))
    self.dt_bias = nn.Parameter(torch.zeros(H * d))
    self.norm = nn.Parameter(torch.ones(e))
    conv = (-0.5, 0.5)
    self.init_ranges = {"q_conv": conv, "k_conv": conv, "v_conv": conv, "a_log": (0.0, 1.0),
                        "dt_bias": (-5.0, -2.0), "norm": (0.8, 1.2)}

  @staticmethod
  def state_spec(p: dict, capacity: int, dtype: torch.dtype, device) -> StateSpec:
    H, G, d, e = p["heads"], p["kv_heads"], p["dim"], p["vdim"]
    return {"s": ((H, e, mo.row_pad(d)), torch.float32),
            # the convolutions' last inputs, position p in row p % taps
            "conv": ((p["conv"], 2 * G * d + H * e), dtype)}

  @staticmethod
  def param_count(dim: int, p: dict) -> int:
    H, G, d, e = p["heads"], p["kv_heads"], p["dim"], p["vdim"]
    ra, rg = p["decay_rank"], p["gate_rank"]
    channels = 2 * G * d + H * e
    return dim * (channels + ra + rg + H + H * e) + channels * p["conv"] + H * d * (ra + 1) + H * e * rg + H + e

  def forward(self, h, proj, at, state, rows, **out):
    pre_decay = self.decay_up(proj[..., at["a1"]:at["a1"] + self.ranks[0]])
    pre_gate = self.gate_up(proj[..., at["g1"]:at["g1"] + self.ranks[1]])
    return mo.delta_rule(proj, [at[n] for n in ("q", "k", "v", "b")], self.H, self.G, self.dim, self.vdim,
                         (self.q_conv, self.k_conv, self.v_conv), pre_decay, pre_gate, self.a_log, self.dt_bias,
                         self.norm, self.eps, state, rows, **out)


class BranchMixer(nn.Module):
  """Branches side by side on one input: weight_0 * branch_0 + ... through a
  fused input projection and a fused output projection."""

  def __init__(self, dim: int, branches: List[Tuple[str, nn.Module, float]]):
    super().__init__()
    self.names = [n for n, _, _ in branches]
    self.weights = [float(s) for _, _, s in branches]
    self.branches = nn.ModuleDict({n: b for n, b, _ in branches})
    # parts start at multiples of 8 (vector loads), the whole at a multiple of
    # 128 rows (the packed decode GEMM's tile); the gaps are zero weights
    self.at: Dict[str, Dict[str, int]] = {}
    n = 0
    for name, branch, _ in branches:
      self.at[name] = {}
      for part, rows in branch.parts:
        self.at[name][part] = n
        n = _up(n + rows, 8)
    self.in_proj = XotLinear(dim, _up(n, 128), bias=False)
    self.out_at, k = {}, 0
    for name, branch, _ in branches:
      self.out_at[name] = k
      k = _up(k + branch.width, 8)
    self.out_width = _up(k, 64)
    self.gapless = self.out_width == sum(b.width for _, b, _ in branches)
    self.o_proj = XotLinear(self.out_width, dim, bias=False)

  def forward(self, h, state, rows):
    proj = self.in_proj(h)
    if proj.is_cuda and not (torch.is_grad_enabled() and proj.requires_grad):
      # zero columns between branches must hold numbers, not leftovers
      new = torch.empty if self.gapless else torch.zeros
      act = new(*proj.shape[:-1], self.out_width, dtype=proj.dtype, device=proj.device)
      for i, name in enumerate(self.names):
        self.branches[name](h, proj, self.at[name], state[i], rows,
                            out=act, out_at=self.out_at[name], out_scale=self.weights[i])
    else:
      pieces, n = [], 0
      for i, name in enumerate(self.names):
        o = self.branches[name](h, proj, self.at[name], state[i] if state is not None else None, rows,
                                out_scale=self.weights[i])
        pieces += [o.new_zeros(*o.shape[:-1], self.out_at[name] - n), o]
        n = self.out_at[name] + o.shape[-1]
      pieces.append(proj.new_zeros(*proj.shape[:-1], self.out_width - n))
      act = torch.cat(pieces, dim=-1)
    return self.o_proj(act)


class ParallelMixer(BranchMixer):
  """Window attention (left) and a gated delta rule (right) on one input."""

  BRANCHES = (("left", WindowBiasAttention), ("right", GatedDeltaRule))

  def __init__(self, dim: int, p: dict, eps: float):
    super().__init__(dim, [(n, c(dim, p[n], eps), p[n + "_scale"]) for n, c in self.BRANCHES])

  @classmethod
  def state_spec(cls, p: dict, capacity: int, dtype: torch.dtype, device) -> List[StateSpec]:
    return [c.state_spec(p[n], capacity, dtype, device) for n, c in cls.BRANCHES]

  @classmethod
  def param_count(cls, dim: int, p: dict) -> int:
    return sum(c.param_count(dim, p[n]) for n, c in cls.BRANCHES)

  @classmethod
  def fill_sizes(cls, p: dict, shapes: Dict[str, tuple], prefix: str):
    """Sizes that only the checkpoint's tensors give."""
    for n, part, key, name, axis in (("left", "rel", "buckets", "bias rows", 0),
                                     ("right", "a1", "decay_rank", "decay rank", 0),
                                     ("right", "g1", "gate_rank", "gate rank", 0)):
      _fill(p[n], key, shapes, f"{prefix}{n}.{part}", axis, name)

  def key_map(self, src: str, dst: str) -> Dict[str, str]:
    """Checkpoint tensor -> parameter of this module (models/weights.py)."""
    m = {}
    for name in self.names:
      for part, _ in self.branches[name].parts:
        m[f"{src}{name}.{part}"] = f"{dst}in_proj.weight@{self.at[name][part]}"
      m[f"{src}{name}.o"] = f"{dst}o_proj.weight@0,{self.out_at[name]}"
    left, right = (f"{dst}branches.{n}." for n in ("left", "right"))
    for theirs, ours in (("q.norm", "q_norm"), ("k.norm", "k_norm"), ("rel", "rel")):
      m[f"{src}left.{theirs}"] = left + ours
    for theirs, ours in (("q.conv", "q_conv"), ("k.conv", "k_conv"), ("v.conv", "v_conv"), ("A_log", "a_log"),
                         ("dt_bias", "dt_bias"), ("norm", "norm"), ("a2", "decay_up.weight"), ("g2", "gate_up.weight")):
      m[f"{src}right.{theirs}"] = right + ours
    return m


class WKVMixer(nn.Module):
  """RWKV-style time mixing: every projection reads its own blend of the
  current and the previous token, a decayed fp32 outer-product memory with a
  bonus for the current token, an RMS norm per head and a silu gate."""

  MIX = ("r", "k", "v", "g", "w")

  def __init__(self, dim: int, p: dict, eps: float):
    super().__init__()
    self.H, self.dim, self.eps = p["heads"], p["dim"], eps
    n = self.H * self.dim
    self.mu = nn.Parameter(torch.zeros(len(self.MIX), dim))
    for name in ("r", "k", "v", "g"):
      setattr(self, f"{name}_proj", XotLinear(dim, n, bias=False))
    self.decay_down = XotLinear(dim, p["decay_rank"], bias=False)
    self.decay_up = XotLinear(p["decay_rank"], n, bias=False)
    self.w0 = nn.Parameter(torch.zeros(n))
    self.u = nn.Parameter(torch.zeros(self.H, self.dim))
    self.norm = nn.Parameter(torch.ones(n))
    self.o_proj = XotLinear(n, dim, bias=False)
    self.init_ranges = {"mu": (0.0, 1.0), "w0": (-6.0, -1.0), "u": (-0.5, 0.5), "norm": (0.8, 1.2)}

  @staticmethod
  def state_spec(p: dict, capacity: int, dtype: torch.dtype, device) -> List[StateSpec]:
    H, d = p["heads"], p["dim"]
    return [{"s": ((H, d, mo.row_pad(d)), torch.float32), "shift": ((2, p["width"]), dtype)}]

  @staticmethod
  def param_count(dim: int, p: dict) -> int:
    n, r = p["heads"] * p["dim"], p["decay_rank"]
    return 5 * dim * n + r * (dim + n) + 5 * dim + 3 * n

  @staticmethod
  def fill_sizes(p: dict, shapes: Dict[str, tuple], prefix: str):
    _fill(p, "decay_rank", shapes, f"{prefix}w1", 0, "decay rank")

  def key_map(self, src: str, dst: str) -> Dict[str, str]:
    m = {f"{src}mu.{n}": f"{dst}mu@{i}" for i, n in enumerate(self.MIX)}
    for n in ("r", "k", "v", "g", "o"):
      m[f"{src}{n}"] = f"{dst}{n}_proj.weight"
    m[f"{src}w1"], m[f"{src}w2"] = f"{dst}decay_down.weight", f"{dst}decay_up.weight"
    m[f"{src}w0"], m[f"{src}u"], m[f"{src}norm"] = f"{dst}w0", f"{dst}u", f"{dst}norm"
    return m

  def forward(self, h, state, rows):
    S, shift = state[0] if state is not None else (None, None)
    r, k, v, g, w = mo.token_shift(h, self.mu, shift, rows)
    pre = self.decay_up(mo.tanh(self.decay_down(w)))
    o = mo.wkv(self.r_proj(r), self.k_proj(k), self.v_proj(v), self.g_proj(g), pre,
               self.w0, self.u, self.norm, self.H, self.dim, self.eps, S, rows)
    return self.o_proj(o)


def _fill(p: dict, key: str, shapes: Dict[str, tuple], tensor: str, axis: int, what: str):
  if tensor in shapes:
    p[key] = shapes[tensor][axis]
  elif key not in p:
    raise ValueError(f"no tensor {tensor} and no '{key}' in the configuration: {what} unknown")


class ChunkAttention(nn.Module):
  """GQA attention within chunks of the sequence, counted from its start: an
  RMS norm per head on q and k, no rotation, a bias that falls linearly with
  the distance, a learned sink per head. With `v_mix`, all but the first such
  layer blend their values with the first one's for the same token."""

  hip = ("_hip_attn",)

  def __init__(self, dim: int, p: dict, eps: float):
    super().__init__()
    self.H, self.G, self.dim, self.vdim = p["heads"], p["kv_heads"], p["dim"], p["vdim"]
    if self.H % self.G:
      raise ValueError(f"{self.H} query heads do not divide into {self.G} key/value heads")
    self.scale, self.chunk, self.eps = float(p["scale"]), int(p["mask"]["size"]), eps
    if self.chunk < 1:
      raise ValueError(f"chunks of {self.chunk} tokens")
    self.shares, self.mixes = bool(p.get("v_first")), bool(p.get("v_mix")) and not p.get("v_first")
    self.parts = [("q", self.H * self.dim), ("k", self.G * self.dim), ("v", self.G * self.vdim)]
    self.width = self.H * self.vdim
    self.q_norm = nn.Parameter(torch.ones(self.dim))
    self.k_norm = nn.Parameter(torch.ones(self.dim))
    self.sink = nn.Parameter(torch.zeros(self.H))
    self.init_ranges = {"q_norm": (0.8, 1.2), "k_norm": (0.8, 1.2), "sink": (-1.0, 1.0)}
    if self.mixes:
      self.v_mix = nn.Parameter(torch.zeros(()))
      self.init_ranges["v_mix"] = (0.3, 0.7)

  @staticmethod
  def state_spec(p: dict, capacity: int, dtype: torch.dtype, device) -> StateSpec:
    # position t lies in row t % chunk: only one chunk of keys is ever read
    return WindowBiasAttention.state_spec(p, capacity, dtype, device)

  @staticmethod
  def param_count(dim: int, p: dict) -> int:
    H, G, d, e = p["heads"], p["kv_heads"], p["dim"], p["vdim"]
    return dim * (H * d + G * d + G * e + H * e) + 2 * d + H

  def forward(self, h, proj, at, state, rows, **out):
    if self.shares:
      rows.carried["values"] = proj[..., at["v"]:at["v"] + self.G * self.vdim]
    mix = (rows.carried["values"], self.v_mix) if self.mixes else None
    return mo.chunk_attn(proj, [at[n] for n, _ in self.parts], self.H, self.G, self.dim, self.vdim, self.q_norm,
                         self.k_norm, self.sink, mix, self.scale, self.eps, self.chunk, state, rows, **out)


def turn_rates(rot: dict) -> List[float]:
  """Radians per position of every pair of turned dimensions. With `scaling`,
  wavelengths beyond original / low are stretched by `factor`, those below
  original / high stay, and the ones between blend."""
  out, s = [], rot.get("scaling")
  for i in range(rot["dims"] // 2):
    f = float(rot["base"]) ** (-2.0 * i / rot["dims"])
    if s is not None:
      turns = s["original"] * f / (2 * math.pi)  # within the original length
      blend = min(1.0, max(0.0, (turns - s["low"]) / (s["high"] - s["low"])))
      f = f * (blend + (1 - blend) / s["factor"])
    out.append(f)
  return out


class Turning(nn.Module):
  """A module with a table of turn rates, which stays in 32-bit whatever the
  model is cast to."""

  def __init__(self):
    super().__init__()
    self.register_buffer("freq", torch.empty(0), persistent=False)

  def rates(self) -> List[float]:
    return turn_rates(self.rot)

  def reset_tables(self, device=None):
    self.freq = torch.tensor(self.rates(), dtype=torch.float32, device=device or self.freq.device)

  def _apply(self, fn, recurse=True):
    super()._apply(fn, recurse)
    if self.freq.dtype != torch.float32:
      self.freq = self.freq.float()
      if self.freq.device.type != "meta":
        self.reset_tables(self.freq.device)
    return self


class LatentAttention(Turning):
  """Latent attention: keys and values of all heads come out of one normed
  latent per token, plus one rotated key part that the heads share. Only these
  two are cached; decode folds the expansion into query and output. With `sink`,
  a learned score per head joins the softmax's denominator; with `gate`, the
  heads' outputs are multiplied with the sigmoid of one more projection."""

  hip = ("_hip_latent", "_hip_attn")

  def __init__(self, dim: int, p: dict, eps: float):
    super().__init__()
    self.H, self.dim, self.rot_dim, self.vdim, self.rank = (p[n] for n in ("heads", "dim", "rot_dim", "vdim", "kv_rank"))
    self.rot, self.scale, self.eps = p["rot"], float(p["scale"]), eps
    if self.rot_dim % 2 or self.rot["dims"] % 2 or self.rot["dims"] > self.rot_dim:
      raise ValueError(f"rotation of {self.rot['dims']} of {self.rot_dim} dimensions")
    self.width = self.H * self.vdim
    self.parts = [("q", self.H * (self.dim + self.rot_dim)), ("dkv", self.rank + self.rot_dim)]
    if p.get("gate"):
      self.parts.append(("g", self.width))
    self.kv_norm = nn.Parameter(torch.ones(self.rank))
    self.kv_up = XotLinear(self.rank, self.H * (self.dim + self.vdim), bias=False)  # all keys, then all values
    self.sink = nn.Parameter(torch.zeros(self.H)) if p.get("sink") else None
    self.init_ranges = {"kv_norm": (0.8, 1.2), "sink": (-1.0, 1.0)}
    self.reset_tables()

  def rates(self) -> List[float]:
    """Pairs that do not rotate have a rate of zero."""
    rates = turn_rates(self.rot)
    return rates + [0.0] * (self.rot_dim // 2 - len(rates))

  @staticmethod
  def state_spec(p: dict, capacity: int, dtype: torch.dtype, device) -> StateSpec:
    R, r = p["kv_rank"], p["rot_dim"]
    if mo.packed_kv(dtype, device):
      # MFMA fragment order of one key/value head, dims padded with zeros
      n = _up(capacity, 32)
      return {"k": ((n // 16, _up(R + r, 32) // 32, 64, 8), dtype), "v": ((_up(R, 16) // 16, n // 32, 64, 8), dtype)}
    return {"k": ((capacity, R + r), dtype), "v": ((capacity, R), dtype)}

  @staticmethod
  def param_count(dim: int, p: dict) -> int:
    H, d, r, e, R = (p[n] for n in ("heads", "dim", "rot_dim", "vdim", "kv_rank"))
    extra = dim * H * e * bool(p.get("gate")) + H * bool(p.get("sink"))
    return dim * (H * (d + r) + R + r + H * e) + R * (H * (d + e) + 1) + extra

  def forward(self, h, proj, at, state, rows, **out):
    return mo.latent_attn(proj, at["q"], at["dkv"], self.H, self.dim, self.rot_dim, self.rank, self.vdim, self.kv_norm,
                          self.kv_up, self.freq, self.scale, self.eps, state, rows, self.sink, at.get("g"), **out)


class RotaryAttention(Turning):
  """GQA attention with rotary positions, causal or over a sliding window that
  keeps the first tokens in sight.

  p: heads, kv_heads, dim, vdim, rot {base, dims, scaling}, scale and
  - mask {size, keep_first}: the window; none: causal
  - softcap: scores become softcap * tanh(score / softcap)
  - pairs: neighbours turn together (else dimensions half the turned ones apart)
  - norm: "before" the rotation, an RMS norm per head with a weight, or "after"
    it, one without
  - values: "own" projection, or the "keys" as projected
  - diff: two maps per head over the same values; the output is the first minus
    lambda times the second, RMS-normed per head and scaled by 1 - diff
  - kv_from: the layer whose cached keys and values this one reads instead of
    having its own; lent: another layer reads this one's; keeps: the layer read
    from is in another shard, so this one caches what travels with the stream
  """

  hip = ("_hip_rotary",)

  def __init__(self, dim: int, p: dict, eps: float):
    super().__init__()
    self.H, self.G, self.dim, self.vdim = p["heads"], p["kv_heads"], p["dim"], p["vdim"]
    self.rot, self.maps = p["rot"], 2 if p.get("diff") is not None else 1
    if self.H % self.G:
      raise ValueError(f"{self.H} query heads do not divide into {self.G} key/value heads")
    if self.rot["dims"] % 2 or self.rot["dims"] > self.dim:
      raise ValueError(f"rotation of {self.rot['dims']} of {self.dim} dimensions")
    if p["values"] == "keys" and (self.vdim != self.dim or self.maps != 1):
      raise ValueError(f"keys of {self.dim} dimensions are no values of {self.vdim}")
    mask = p.get("mask") or {"size": 0, "keep_first": 0}
    if p.get("mask") and mask["size"] < 1:
      raise ValueError(f"window of {mask['size']} tokens")
    self.layer, self.source = p.get("layer"), p.get("kv_from")
    self.lent, self.keeps = bool(p.get("lent")), bool(p.get("keeps"))
    if (self.lent or self.source is not None) and (p.get("mask") or p["values"] == "keys"):
      raise ValueError("only causal attention with values of its own shares them")
    self.rule = mo.AttnRule(
      self.H, self.G, self.dim, self.vdim, self.maps, float(p["scale"]), float(p.get("softcap") or 0.0),
      int(mask["size"]), int(mask.get("keep_first", 0)), bool(p["pairs"]), p["norm"] == "after", eps,
      1.0 - p["diff"] if self.maps == 2 else 1.0)
    q, k = ("q", self.H * self.maps * self.dim), ("k", self.G * self.maps * self.dim)
    self.parts = [q] if self.source is not None else [q, k] if p["values"] == "keys" else [q, k, ("v", self.G * self.vdim)]
    self.width = self.H * self.vdim
    self.init_ranges = {}
    self.q_norm = self.k_norm = None
    if p["norm"] == "before":
      self.q_norm = nn.Parameter(torch.ones(self.dim))
      self.init_ranges["q_norm"] = (0.8, 1.2)
      if self.source is None or self.keeps:
        self.k_norm = nn.Parameter(torch.ones(self.dim))
        self.init_ranges["k_norm"] = (0.8, 1.2)
    if self.maps == 2:
      self.diff = float(p["diff"])
      self.contrast = nn.Parameter(torch.zeros(4, self.dim))  # the vectors of lambda: q1, k1, q2, k2
      self.init_ranges["contrast"] = (-0.1, 0.1)
    self.reset_tables()

  @staticmethod
  def lent_width(p: dict) -> int:
    """Channels of what travels with the stream: keys and values as projected."""
    return _up(2 * p["kv_heads"] * p["dim"], 8) + p["kv_heads"] * p["vdim"]

  @staticmethod
  def state_spec(p: dict, capacity: int, dtype: torch.dtype, device) -> StateSpec:
    if p.get("kv_from") is not None and not p.get("keeps"):
      return {}
    G, d, e, mask = p["kv_heads"], p["dim"], p["vdim"], p.get("mask")
    maps = 2 if p.get("diff") is not None else 1
    # the kept tokens' rows, then a ring of the window's
    n = min(capacity, mask["size"] + mask.get("keep_first", 0)) if mask else capacity
    if mo.packed_kv(dtype, device):
      n = _up(n, 32)  # MFMA fragment order, as for WindowBiasAttention
      return {"k": ((G * maps, n // 16, _up(d, 32) // 32, 64, 8), dtype),
              "v": ((G, _up(e, 16) // 16, n // 32, 64, 8), dtype)}
    return {"k": ((G * maps, n, d), dtype), "v": ((G, n, e), dtype)}

  @staticmethod
  def param_count(dim: int, p: dict) -> int:
    H, G, d, e = p["heads"], p["kv_heads"], p["dim"], p["vdim"]
    maps = 2 if p.get("diff") is not None else 1
    own = 0 if p.get("kv_from") is not None else G * maps * d + (G * e if p["values"] == "own" else 0)
    return dim * (H * maps * d + own + H * e) + (2 * d if p["norm"] == "before" else 0) + (4 * d if maps == 2 else 0)

  def contrast_weight(self):
    """lambda as a 32-bit tensor; outside of training kept with the module."""
    if self.maps == 1:
      return None

    def value():
      q1, k1, q2, k2 = self.contrast.float()
      return torch.exp((q1 * k1).sum()) - torch.exp((q2 * k2).sum()) + self.diff
    if torch.is_grad_enabled() and self.contrast.requires_grad:
      return value()
    key = (self.contrast.data_ptr(), self.contrast._version)
    if getattr(self, "_lambda_key", None) != key:
      self._lambda, self._lambda_key = value().reshape(1), key
    return self._lambda

  def forward(self, h, proj, at, state, rows, **out):
    source, k_norm, append = None, self.k_norm, True
    if self.source is None:
      source = (proj, at["k"], at.get("v", at["k"]))
      if self.lent:
        rows.carried[f"kv{self.layer}"] = proj[..., at["k"]:at["v"] + self.G * self.vdim]
    elif self.keeps:
      source = (rows.carried[f"kv{self.source}"].contiguous(), 0, _up(self.G * self.maps * self.dim, 8))
    else:
      state, source, k_norm = rows.kept[self.source]
      append = False
    if self.lent or self.keeps:
      rows.kept[self.layer if self.lent else self.source] = (state, source, k_norm)
    return mo.rotary_attn(proj, at["q"], source, self.rule, self.q_norm, k_norm, self.freq, self.contrast_weight(), state,
                          rows, append, **out)


class GatedLinearUnit(nn.Module):
  """Recurrent block of a gated linear unit: a short causal convolution, gates
  of recurrence and input through block-diagonal products, an fp32 state per
  channel, and a gelu branch that multiplies the result."""

  RATE = 8.0  # the decay's exponent at an open gate, in softplus(lam)

  hip = ("_hip_lru", "_hip_scan",)

  def __init__(self, dim: int, p: dict, eps: float):
    super().__init__()
    self.width, self.blocks = p["width"], p["blocks"]
    if self.width % self.blocks:
      raise ValueError(f"{self.width} channels do not divide into {self.blocks} blocks")
    W, n = self.width, self.width // self.blocks
    self.parts = [("y", W), ("x", W)]
    self.in_bias = nn.Parameter(torch.zeros(2, W))
    self.conv = nn.Parameter(torch.zeros(W, p["conv"]))
    self.conv_bias = nn.Parameter(torch.zeros(W))
    self.gates = nn.Parameter(torch.zeros(2, self.blocks, n, n))  # of the recurrence, of the input
    self.gate_bias = nn.Parameter(torch.zeros(2, self.blocks, n))
    self.lam = nn.Parameter(torch.zeros(W))
    self.init_ranges = {"in_bias": (-0.1, 0.1), "conv": (-0.5, 0.5), "conv_bias": (-0.1, 0.1), "gate_bias": (-1.0, 1.0),
                        "lam": (-6.0, -2.0)}

  @staticmethod
  def state_spec(p: dict, capacity: int, dtype: torch.dtype, device) -> StateSpec:
    return {"s": ((p["width"],), torch.float32),
            # the convolution's last inputs, position t in row t % taps
            "conv": ((p["conv"], p["width"]), dtype)}

  @staticmethod
  def param_count(dim: int, p: dict) -> int:
    W, n = p["width"], p["width"] // p["blocks"]
    return W * (3 * dim + 2 * n + p["conv"] + 6)

  def forward(self, h, proj, at, state, rows, **out):
    return mo.gated_unit(proj, at["y"], at["x"], self.in_bias, self.conv, self.conv_bias, self.gates, self.gate_bias,
                         self.lam, self.RATE, state, rows, **out)


class MatrixMemory(nn.Module):
  """Matrix memory with exponential gates (the mLSTM of xLSTM): per head an fp32
  state that decays by a forget gate and takes in the outer product of key and
  value by an input gate, both kept as logarithms (capped) relative to a running
  maximum; the read-out is divided by what the queries find of the keys, then
  RMS-normed per head, weighted and gated."""

  hip = ("_hip_mlstm",)

  def __init__(self, dim: int, p: dict, eps: float):
    super().__init__()
    self.H, self.dim, self.vdim, self.cap, self.eps = p["heads"], p["dim"], p["vdim"], float(p["gate_cap"]), eps
    if self.cap <= 0:
      raise ValueError(f"gates capped at {self.cap}")
    self.width = self.H * self.vdim
    self.parts = [("q", self.H * self.dim), ("k", self.H * self.dim), ("v", self.width), ("g", self.width),
                  ("i", self.H), ("f", self.H)]
    self.gate_bias = nn.Parameter(torch.zeros(2, self.H))  # of the input gate, of the forget gate
    self.norm = nn.Parameter(torch.ones(self.width))
    self.init_ranges = {"gate_bias": (1.0, 5.0), "norm": (0.8, 1.2)}

  @staticmethod
  def state_spec(p: dict, capacity: int, dtype: torch.dtype, device) -> StateSpec:
    # a row of key channels per value channel; the last one sums the keys alone
    return {"s": ((p["heads"], p["vdim"] + 1, mo.row_pad(p["dim"])), torch.float32),
            "m": ((p["heads"],), torch.float32)}

  @staticmethod
  def param_count(dim: int, p: dict) -> int:
    H, d, e = p["heads"], p["dim"], p["vdim"]
    return dim * H * (2 * d + 3 * e + 2) + H * (e + 2)

  def forward(self, h, proj, at, state, rows, **out):
    return mo.matrix_memory(proj, [at[n] for n, _ in self.parts], self.H, self.dim, self.vdim, self.gate_bias, self.cap,
                            self.norm, self.eps, state, rows, **out)


class SelectiveScan(nn.Module):
  """Selective state space: short causal convolution and silu, step sizes
  through a low-rank pair, an fp32 state [inner, state], skip and silu gate."""

  hip = ("_hip_scan",)

  def __init__(self, dim: int, p: dict, eps: float):
    super().__init__()
    self.inner, self.n, self.rank = p["inner"], p["state"], p["dt_rank"]
    self.parts = [("in", 2 * self.inner)]  # what is scanned, then its gate
    self.width = self.inner
    self.conv = nn.Parameter(torch.zeros(self.inner, p["conv"]))
    self.conv_bias = nn.Parameter(torch.zeros(self.inner))
    self.x_proj = XotLinear(self.inner, self.rank + 2 * self.n, bias=False)
    self.dt_proj = XotLinear(self.rank, self.inner, bias=False)
    self.dt_bias = nn.Parameter(torch.zeros(self.inner))
    self.a_log = nn.Parameter(torch.zeros(self.inner, self.n))
    self.skip = nn.Parameter(torch.ones(self.inner))
    self.init_ranges = {"conv": (-0.5, 0.5), "conv_bias": (-0.1, 0.1), "dt_bias": (-5.0, -2.0), "a_log": (0.0, 2.5),
                        "skip": (0.8, 1.2)}

  @staticmethod
  def state_spec(p: dict, capacity: int, dtype: torch.dtype, device) -> StateSpec:
    return {"s": ((p["inner"], p["state"]), torch.float32),
            # the convolution's last inputs, position t in row t % taps
            "conv": ((p["conv"], p["inner"]), dtype)}

  @staticmethod
  def param_count(dim: int, p: dict) -> int:
    inner, n, rank = p["inner"], p["state"], p["dt_rank"]
    return inner * (3 * dim + p["conv"] + 2 * rank + 3 * n + 3)

  def forward(self, h, proj, at, state, rows, **out):
    s, ring = state if state is not None else (None, None)
    x = mo.conv_silu(proj, at["in"], self.conv, self.conv_bias, ring, rows)
    low = self.x_proj(x)
    pre = self.dt_proj(low[..., :self.rank])
    return mo.selective_scan(x, pre, low, self.rank, self.rank + self.n, proj, at["in"] + self.inner, self.a_log,
                             self.dt_bias, self.skip, s, rows, **out)


class SingleMixer(BranchMixer):
  """One branch between its fused input projection and its output projection."""

  BRANCH: type
  TENSORS: Dict[str, str]  # checkpoint tensor -> parameter of the branch

  def __init__(self, dim: int, p: dict, eps: float):
    super().__init__(dim, [("only", self.BRANCH(dim, p, eps), 1.0)])

  @classmethod
  def state_spec(cls, p: dict, capacity: int, dtype: torch.dtype, device) -> List[StateSpec]:
    return [cls.BRANCH.state_spec(p, capacity, dtype, device)]

  @classmethod
  def param_count(cls, dim: int, p: dict) -> int:
    return cls.BRANCH.param_count(dim, p)

  def key_map(self, src: str, dst: str) -> Dict[str, str]:
    m = {f"{src}{part}": f"{dst}in_proj.weight@{at}" for part, at in self.at["only"].items()}
    m[f"{src}o"] = f"{dst}o_proj.weight@0,0"
    own = dict(self.branches["only"].named_parameters())
    m.update({src + theirs: f"{dst}branches.only.{ours}" for theirs, ours in self.TENSORS.items()
              if ours in own})
    return m


class ChunkAttentionMixer(SingleMixer):
  BRANCH = ChunkAttention
  TENSORS = {"q.norm": "q_norm", "k.norm": "k_norm", "sink": "sink", "vmix": "v_mix"}


class LatentAttentionMixer(SingleMixer):
  BRANCH = LatentAttention
  TENSORS = {"dkv.norm": "kv_norm", "sink": "sink"}

  def key_map(self, src: str, dst: str) -> Dict[str, str]:
    own = self.branches["only"]
    up = f"{dst}branches.only.kv_up.weight"
    return {**super().key_map(src, dst), f"{src}uk": f"{up}@0", f"{src}uv": f"{up}@{own.H * own.dim}"}


class MatrixMemoryMixer(SingleMixer):
  BRANCH = MatrixMemory
  TENSORS = {"norm": "norm"}

  def key_map(self, src: str, dst: str) -> Dict[str, str]:
    m = super().key_map(src, dst)
    for i, gate in enumerate(("i", "f")):
      m[f"{src}{gate}.b"] = f"{dst}branches.only.gate_bias@{i}"
    return m


class SelectiveScanMixer(SingleMixer):
  BRANCH = SelectiveScan
  TENSORS = {"conv": "conv", "conv.b": "conv_bias", "x": "x_proj.weight", "dt": "dt_proj.weight", "dt.b": "dt_bias",
             "A_log": "a_log", "D": "skip"}


class KeptAttentionMixer(SingleMixer):
  BRANCH = RotaryAttention
  TENSORS = {"q.norm": "q_norm", "k.norm": "k_norm"}


class DifferenceAttentionMixer(KeptAttentionMixer):
  def key_map(self, src: str, dst: str) -> Dict[str, str]:
    m, own = super().key_map(src, dst), self.branches["only"]
    for i, n in enumerate(("lq1", "lk1", "lq2", "lk2")):
      m[src + n] = f"{dst}branches.only.contrast@{i}"
    if own.keeps:  # the norm of the keys it caches is the other layer's
      del m[f"{src}k.norm"]
      m[f"l{own.source}.mix.k.norm"] = f"{dst}branches.only.k_norm"
    return m


class GatedLinearUnitMixer(SingleMixer):
  BRANCH = GatedLinearUnit
  TENSORS = {"conv": "conv", "conv.b": "conv_bias", "lam": "lam"}

  def key_map(self, src: str, dst: str) -> Dict[str, str]:
    m, own = super().key_map(src, dst), f"{dst}branches.only."
    for i, (branch, gate) in enumerate((("y", "ra"), ("x", "ri"))):
      m[f"{src}{branch}.b"] = f"{own}in_bias@{i}"
      m[f"{src}{gate}"], m[f"{src}{gate}.b"] = f"{own}gates@{i}", f"{own}gate_bias@{i}"
    return m


MIXERS = {"kept_attention": KeptAttentionMixer, "difference_attention": DifferenceAttentionMixer,
          "rglru": GatedLinearUnitMixer, "parallel": ParallelMixer, "wkv": WKVMixer, "chunk_attention": ChunkAttentionMixer,
          "latent_attention": LatentAttentionMixer, "mamba1": SelectiveScanMixer, "mlstm": MatrixMemoryMixer}
