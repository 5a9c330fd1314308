"""Sparse feed-forward of small experts, computed as grouped products.

Sigmoid scores with a correction that only chooses, group-limited top-k and
scaled weights, or a softmax over the chosen logits; a gated activation with
clipped inputs; a gated shared expert; every constant is a parameter. The experts' weights lie in two
stacked tensors, padded with zeros to what the kernels walk (ops/hip/
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
  """p: {"expert": {ff, limit, alpha, plus}, "router": {experts, top, weights,
  scale, groups: {count, keep}}, "shared": {ff} or None}. The router's weights
  are "sigmoid" scores (chosen with a learned correction) or the "softmax" of
  the chosen logits. A shared expert, which every token uses with a sigmoid
  gate of its own, is cut into pieces of the experts' width: experts that are
  always chosen, all with that gate."""

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
    wide = _up(self.ff, 64)
    self.shared_ff = shared["ff"] if shared else 0
    self.pieces = -(-self.shared_ff // wide)
    self.rule = mo.Routing(r["top"], groups["count"], groups["keep"], float(r.get("scale", 1.0)), weights == "softmax",
                           self.pieces)
    e = p["expert"]
    self.act = (float(e.get("alpha", ALPHA)), float(e["limit"]), float(e.get("plus", PLUS)))
    # a row for the shared expert's gate follows the router's own
    self.router = nn.Parameter(torch.zeros(self.E + bool(self.pieces), dim))
    self.correction = None if self.rule.softmax else nn.Parameter(torch.zeros(self.E))
    self.gate_up = nn.Parameter(torch.zeros(self.E + self.pieces, 2, wide, _up(dim, 64)))
    self.down = nn.Parameter(torch.zeros(self.E + self.pieces, _up(dim, 16), wide))
    self.init_ranges = {} if self.rule.softmax else {"correction": (-0.1, 0.1)}

  @torch.no_grad()
  def zero_padding(self):
    """After random initialization: the kernels count on zeros there."""
    self.gate_up[..., self.dim:] = 0
    self.down[:, self.dim:] = 0
    for e in range(self.E + self.pieces):
      ff = self.ff if e < self.E else min(self.down.shape[-1], self.shared_ff - (e - self.E) * self.down.shape[-1])
      self.gate_up[e, :, ff:] = 0
      self.down[e, :, ff:] = 0

  @staticmethod
  def param_count(dim: int, p: dict) -> int:
    r, shared = p["router"], p.get("shared")
    n = r["experts"] * (3 * dim * p["expert"]["ff"] + dim + (r.get("weights", "sigmoid") == "sigmoid"))
    return n + (dim * (3 * shared["ff"] + 1) if shared else 0)

  def key_map(self, src: str, dst: str) -> Dict[str, str]:
    m = {f"{src}router": f"{dst}router@0"}
    if self.correction is not None:
      m[f"{src}correction"] = f"{dst}correction"
    for e in range(self.E):
      m[f"{src}e{e}.gate"] = f"{dst}gate_up@{e},0"
      m[f"{src}e{e}.up"] = f"{dst}gate_up@{e},1"
      m[f"{src}e{e}.down"] = f"{dst}down@{e}"
    if self.pieces:
      wide = self.down.shape[-1]
      cuts = [(self.E + i, i * wide, min(self.shared_ff, (i + 1) * wide)) for i in range(self.pieces)]
      m[f"{src}shared.sg"] = f"{dst}router@{self.E}"
      m[f"{src}shared.gate"] = ";".join(f"{dst}gate_up@{e},0<0,{lo}:{hi}" for e, lo, hi in cuts)
      m[f"{src}shared.up"] = ";".join(f"{dst}gate_up@{e},1<0,{lo}:{hi}" for e, lo, hi in cuts)
      m[f"{src}shared.down"] = ";".join(f"{dst}down@{e}<1,{lo}:{hi}" for e, lo, hi in cuts)
    return m

  def forward(self, h):
    """The mixture [.., dim], or (on the HIP path) its rows for mo.add_norm."""
    return mo.expert_mixture(h, self.router, self.correction, self.gate_up, self.down, self.ff, self.rule,
                             self.act)
