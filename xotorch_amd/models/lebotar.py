"""Lebotar decoder (models/layered.py): attention within chunks of the
sequence (whose layers may share values), latent attention, and selective
state spaces, each with a sparse feed-forward or none. Pre-norm with weights
stored around zero; every sublayer's output is scaled before it joins the fp32
stream, in the same kernel that norms the stream for the next sublayer.
"""
from __future__ import annotations

import copy
from typing import Dict, List

import torch
import torch.nn as nn

from xotorch_amd.models.config import _DTYPE_MAP, LayerSpec, ModelConfig
from xotorch_amd.models.experts import GroupedExperts
from xotorch_amd.models.layered import LayeredModel, layered_key_map, max_positions
from xotorch_amd.models.mixers import MIXERS
from xotorch_amd.ops import mixer_ops as mo
from xotorch_amd.shard import Shard

# layer type in config.json -> mixer
TYPES = {"attention": "chunk_attention", "latent_attention": "latent_attention", "mamba1": "mamba1"}


def lebotar_config(raw: dict, model_id: str, shapes: Dict[str, tuple]) -> ModelConfig:
  specs: List[LayerSpec] = []
  shared = 0  # width of the values that later layers mix in
  for i, entry in enumerate(raw["layers"]):
    kind = entry["type"]
    if kind not in TYPES:
      raise ValueError(f"layer {i}: unknown mixer {kind!r}")
    params = copy.deepcopy(entry["mixer"])
    if params.get("v_mix"):
      width = params["kv_heads"] * params["vdim"]
      params["v_first"] = not shared
      if shared and width != shared:
        raise ValueError(f"layer {i}: {width} value channels cannot mix with an earlier layer's {shared}")
      shared = width
    mlp = entry.get("mlp")
    if mlp is not None and mlp["kind"] != "moe":
      raise ValueError(f"layer {i}: unknown feed-forward {mlp['kind']!r}")
    specs.append(LayerSpec(TYPES[kind], params, moe=copy.deepcopy(mlp)))
  moes = [s.moe for s in specs if s.moe is not None]
  return ModelConfig(
    model_id=model_id, model_type="lebotar", vocab_size=raw["vocab"], dim=raw["width"], n_layers=len(specs),
    norm_eps=float(raw["norm"]["eps"]), max_seq_len=max_positions(raw), layer_specs=specs,
    residual_mult=float(raw["residual_mult"]), carried={"values": shared} if shared else {},
    n_experts=max((m["router"]["experts"] for m in moes), default=0),
    moe_intermediate_dim=max((m["expert"]["ff"] for m in moes), default=0),
    intermediate_dim=max((m["expert"]["ff"] for m in moes), default=0),
    torch_dtype=_DTYPE_MAP.get(raw.get("torch_dtype", "bfloat16"), torch.bfloat16),
    bos_token_id=raw.get("bos_token_id"), eos_token_id=raw.get("eos_token_id"),
  )


class LebotarLayer(nn.Module):
  def __init__(self, cfg: ModelConfig, spec: LayerSpec):
    super().__init__()
    self.eps, self.mult = cfg.norm_eps, cfg.residual_mult
    norms = ("norm1", "norm2") if spec.moe is not None else ("norm1",)
    for n in norms:
      self.register_parameter(n, nn.Parameter(torch.zeros(cfg.dim)))
    self.init_ranges = {n: (-0.2, 0.2) for n in norms}
    self.mix = MIXERS[spec.mixer](cfg.dim, spec.params, cfg.norm_eps)
    self.mlp = GroupedExperts(cfg.dim, spec.moe) if spec.moe is not None else None

  def step(self, x, h, cache, rows, after):
    y = self.mix(h, cache, rows)
    x, h = mo.add_norm(y, x, self.mult, self.norm2 if self.mlp is not None else after, self.eps)
    if self.mlp is not None:
      x, h = mo.add_norm(self.mlp(h), x, self.mult, after, self.eps)
    return x, h

  def key_map(self, src: str, dst: str) -> Dict[str, str]:
    m = self.mix.key_map(src + "mix.", dst + "mix.")
    m[src + "norm1"] = dst + "norm1"
    if self.mlp is not None:
      m[src + "norm2"] = dst + "norm2"
      m.update(self.mlp.key_map(src + "mlp.", dst + "mlp."))
    return m


class LebotarModel(LayeredModel):
  def make_layer(self, cfg: ModelConfig, spec: LayerSpec, place: int) -> nn.Module:
    return LebotarLayer(cfg, spec)


def key_map_lebotar(shard: Shard, cfg: ModelConfig) -> Dict[str, str]:
  return layered_key_map(LebotarModel, shard, cfg)
