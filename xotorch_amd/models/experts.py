"""Sparse feed-forward of small experts, computed as grouped products.

Sigmoid scores (with or without a correction that only chooses), group-limited
top-k and scaled weights, or a softmax over the chosen logits, which multiply an
expert's output or its input; a gated activation with clipped inputs or a plain
one; a shared expert, gated or not; every constant is a parameter. The experts'
weights lie in two stacked tensors, padded with zeros to what the kernels walk (ops/hip/
expert_ops.hip), so a step is a handful of launches with static shapes and the
host never waits for a count.
"""
from __future__ import annotations

from typing import Dict

import torch
import torch.nn as nn

from xotorch_amd.ops import mixer_ops as mo

ALPHA = 1.702  # slope of the gate's sigmoid
PLUS = 1.0     # added to the linear half


def _up(n: int, to: int) -> int:
  return -(-n // to) * to


class GroupedExperts(nn.Module):
  """p: {"expert": {ff, act, limit, alpha, plus}, "router": {experts, top, weights,
  scale, corrected, applied, groups: {count, keep}}, "shared": {ff, gated} or
  None}. act: "gated" (the default) or "relu2", the square of relu without a
  gate. The router's weights are "sigmoid" scores (chosen with a learned
  correction unless `corrected` is false) or the "softmax" of the chosen logits;
  they are applied to the experts' "output" (the default) or "input". A shared
  expert, which every token uses, is cut into pieces of the experts' width:
  experts that are always chosen, all with the weight of a sigmoid gate of their
  own or, not `gated`, of one."""

  hip = ("_hip_experts",)

  def __init__(self, dim: int, p: dict):
    super().__init__()
    r, shared = p["router"], p.get("shared")
    groups = r.get("groups") or {"count": 1, "keep": 1}
    self.dim, self.ff, self.E = dim, p["expert"]["ff"], r["experts"]
    if self.E % groups["count"]:
      raise ValueError(f"{self.E} experts do not divide into {groups['count']} groups")
    if r["top"] > groups["keep"] * (self.E // groups["count"]):
      raise ValueError(f"{r['top']} experts cannot come from {groups['keep']} of {groups['count']} groups")
    weights = r.get("weights", "sigmoid")
    if weights not in ("sigmoid", "softmax"):
      raise ValueError(f"unknown router weights {weights!r}")
    if r.get("applied", "output") not in ("output", "input"):
      raise ValueError(f"router weights applied to the {r['applied']!r}")
    wide = _up(self.ff, 64)
    self.shared_ff = shared["ff"] if shared else 0
    self.pieces = -(-self.shared_ff // wide)
    self.shared_gate = bool(self.pieces) and shared.get("gated", True)
    self.rule = mo.Routing(r["top"], groups["count"], groups["keep"], float(r.get("scale", 1.0)), weights == "softmax",
                           self.pieces, self.shared_gate, r.get("applied") == "input")
    e = p["expert"]
    self.gated = e.get("act", "gated") == "gated"
    if self.gated:
      self.act = mo.GatedAct(float(e.get("alpha", ALPHA)), float(e["limit"]), float(e.get("plus", PLUS)))
    elif e["act"] == "relu2":
      self.act = mo.RELU2
    else:
      raise ValueError(f"unknown activation {e['act']!r}")
    # a row for the shared expert's gate follows the router's own
    self.router = nn.Parameter(torch.zeros(self.E + self.shared_gate, dim))
    corrected = not self.rule.softmax and r.get("corrected", True)
    self.correction = nn.Parameter(torch.zeros(self.E)) if corrected else None
    up = nn.Parameter(torch.zeros(self.E + self.pieces, *((2,) if self.gated else ()), wide, _up(dim, 64)))
    self.register_parameter("gate_up" if self.gated else "up", up)
    self.down = nn.Parameter(torch.zeros(self.E + self.pieces, _up(dim, 16), wide))
    self.init_ranges = {"correction": (-0.1, 0.1)} if corrected else {}

  @property
  def first(self):
    """Weights of the first product."""
    return self.gate_up if self.gated else self.up

  @torch.no_grad()
  def zero_padding(self):
    """After random initialization: the kernels count on zeros there."""
    self.first[..., self.dim:] = 0
    self.down[:, self.dim:] = 0
    for e in range(self.E + self.pieces):
      ff = self.ff if e < self.E else min(self.down.shape[-1], self.shared_ff - (e - self.E) * self.down.shape[-1])
      self.first[e, ..., ff:, :] = 0
      self.down[e, :, ff:] = 0

  @staticmethod
  def param_count(dim: int, p: dict) -> int:
    r, shared = p["router"], p.get("shared")
    products = 3 if p["expert"].get("act", "gated") == "gated" else 2
    corrected = r.get("weights", "sigmoid") == "sigmoid" and r.get("corrected", True)
    n = r["experts"] * (products * dim * p["expert"]["ff"] + dim + corrected)
    return n + (dim * (products * shared["ff"] + shared.get("gated", True)) if shared else 0)

  def key_map(self, src: str, dst: str) -> Dict[str, str]:
    m = {f"{src}router": f"{dst}router@0"}
    if self.correction is not None:
      m[f"{src}correction"] = f"{dst}correction"
    parts = {"gate": "gate_up@{},0", "up": "gate_up@{},1"} if self.gated else {"up": "up@{}"}
    for e in range(self.E):
      for theirs, ours in parts.items():
        m[f"{src}e{e}.{theirs}"] = dst + ours.format(e)
      m[f"{src}e{e}.down"] = f"{dst}down@{e}"
    if self.pieces:
      wide = self.down.shape[-1]
      cuts = [(self.E + i, i * wide, min(self.shared_ff, (i + 1) * wide)) for i in range(self.pieces)]
      if self.shared_gate:
        m[f"{src}shared.sg"] = f"{dst}router@{self.E}"
      for theirs, ours in parts.items():
        m[f"{src}shared.{theirs}"] = ";".join(f"{dst}{ours.format(e)}<0,{lo}:{hi}" for e, lo, hi in cuts)
      m[f"{src}shared.down"] = ";".join(f"{dst}down@{e}<1,{lo}:{hi}" for e, lo, hi in cuts)
    return m

  def forward(self, h):
    """The mixture [.., dim], or (on the HIP path) its rows for mo.add_norm."""
    return mo.expert_mixture(h, self.router, self.correction, self.first, self.down, self.ff, self.rule, self.act)
