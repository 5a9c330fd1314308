"""Didipel decoder (models/layered.py): window attention and a gated delta rule
side by side, or RWKV-style time mixing; a dense SwiGLU feed-forward or none;
norms before AND after each sublayer with weights stored around zero. One
fused kernel adds a sublayer's normed output to the stream and norms the
stream for the next sublayer. State per slot is constant in the sequence
length.
"""
from __future__ import annotations

import copy
from typing import Dict, List

import torch
import torch.nn as nn

from xotorch_amd.models.config import _DTYPE_MAP, LayerSpec, ModelConfig
from xotorch_amd.models.layered import LayeredModel, layered_key_map, max_positions
from xotorch_amd.models.llama import MLP
from xotorch_amd.models.mixers import MIXERS
from xotorch_amd.ops import mixer_ops as mo
from xotorch_amd.shard import Shard

TYPES = ("parallel", "wkv")


def didipel_config(raw: dict, model_id: str, shapes: Dict[str, tuple]) -> ModelConfig:
  """config.json (and, for sizes it leaves open, the tensor shapes)."""
  specs: List[LayerSpec] = []
  for i, entry in enumerate(raw["layers"]):
    kind = entry["type"]
    if kind not in TYPES:
      raise ValueError(f"layer {i}: unknown mixer {kind!r}")
    mlp = entry.get("mlp")
    if mlp is not None and mlp["kind"] != "dense":
      raise ValueError(f"layer {i}: unknown feed-forward {mlp['kind']!r}")
    params = copy.deepcopy(entry["mixer"])
    params["width"] = raw["width"]
    MIXERS[kind].fill_sizes(params, shapes, f"l{i}.mix.")
    specs.append(LayerSpec(kind, params, mlp["ff"] if mlp is not None else 0))
  return ModelConfig(
    model_id=model_id, model_type="didipel", vocab_size=raw["vocab"], dim=raw["width"], n_layers=len(specs),
    norm_eps=float(raw["norm"]["eps"]), max_seq_len=max_positions(raw), layer_specs=specs,
    intermediate_dim=max(s.ff for s in specs),
    torch_dtype=_DTYPE_MAP.get(raw.get("torch_dtype", "bfloat16"), torch.bfloat16),
    bos_token_id=raw.get("bos_token_id"), eos_token_id=raw.get("eos_token_id"),
  )


class DenseMLP(MLP):
  """The llama family's SwiGLU block with the activation kernel that takes any
  width and also runs in 32-bit."""

  @staticmethod
  def act(gu):
    return mo.swiglu_packed(gu)


class DenseGeluMLP(DenseMLP):
  """The same block with the tanh form of gelu."""

  def forward(self, x):
    return self.down_proj(mo.gated_packed(self.gate_up_proj(x), "gelu_tanh"))


class DidipelLayer(nn.Module):
  def __init__(self, cfg: ModelConfig, spec: LayerSpec):
    super().__init__()
    self.eps = cfg.norm_eps
    norms = ("norm1", "norm1b") + (("norm2", "norm2b") if spec.ff else ())
    for n in norms:
      self.register_parameter(n, nn.Parameter(torch.zeros(cfg.dim)))
    self.init_ranges = {n: (-0.2, 0.2) for n in norms}
    self.mix = MIXERS[spec.mixer](cfg.dim, spec.params, cfg.norm_eps)
    self.mlp = DenseMLP(cfg, spec.ff) if spec.ff else None

  def step(self, x, h, cache, rows, after):
    y = self.mix(h, cache, rows)
    x, h = mo.sandwich_norm(y, x, self.norm1b, self.norm2 if self.mlp is not None else after, self.eps)
    if self.mlp is not None:
      x, h = mo.sandwich_norm(self.mlp(h), x, self.norm2b, after, self.eps)
    return x, h

  def key_map(self, src: str, dst: str) -> Dict[str, str]:
    m = self.mix.key_map(src + "mix.", dst + "mix.")
    m[src + "norm1"], m[src + "norm1b"] = dst + "norm1", dst + "norm1b"
    if self.mlp is not None:
      m[src + "norm2"], m[src + "norm2b"] = dst + "norm2", dst + "norm2b"
      m[src + "mlp.gate"] = dst + "mlp.gate_up_proj.weight#0"
      m[src + "mlp.up"] = dst + "mlp.gate_up_proj.weight#1"
      m[src + "mlp.down"] = dst + "mlp.down_proj.weight"
    return m


class DidipelModel(LayeredModel):
  def make_layer(self, cfg: ModelConfig, spec: LayerSpec, place: int) -> nn.Module:
    return DidipelLayer(cfg, spec)


def key_map_didipel(shard: Shard, cfg: ModelConfig) -> Dict[str, str]:
  return layered_key_map(DidipelModel, shard, cfg)
