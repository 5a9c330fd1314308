"""Tapupel decoder (models/layered.py): windowed attention with kept first
tokens, differential attention whose later layers may read an earlier one's
keys and values, and gated linear recurrences; a dense SwiGLU feed-forward, a
sparse one with a gated shared expert, or none. Sublayers read the stream
itself; only their outputs are normed, in the kernel that adds them to it.
"""
from __future__ import annotations

import copy
import math
from typing import Dict, List

import torch
import torch.nn as nn

from xotorch_amd.models.config import _DTYPE_MAP, LayerSpec, ModelConfig
from xotorch_amd.models.didipel import DenseMLP
from xotorch_amd.models.experts import GroupedExperts
from xotorch_amd.models.layered import LayeredModel, layered_key_map, max_positions
from xotorch_amd.models.mixers import MIXERS, RotaryAttention
from xotorch_amd.ops import mixer_ops as mo
from xotorch_amd.shard import Shard

# layer type in config.json -> mixer, and what the design fixes about it
TYPES = {
  "attention": ("kept_attention", {"pairs": False, "norm": "after", "values": "keys"}),
  "attention_2": ("difference_attention", {"pairs": True, "norm": "before", "values": "own"}),
  "rglru": ("rglru", {}),
}
SILU = {"alpha": 1.0, "limit": math.inf, "plus": 0.0}  # the gated activation is silu(g) * u


def _feed_forward(i: int, mlp) -> dict:
  if mlp is None:
    return {}
  if mlp["kind"] == "dense":
    return {"ff": mlp["ff"]}
  if mlp["kind"] != "moe":
    raise ValueError(f"layer {i}: unknown feed-forward {mlp['kind']!r}")
  shared = mlp.get("shared")
  return {"moe": {"expert": {"ff": mlp["expert"]["ff"], **SILU}, "shared": dict(shared) if shared else None,
                  "router": {"experts": mlp["router"]["experts"], "top": mlp["router"]["top"], "weights": "softmax"}}}


def tapupel_config(raw: dict, model_id: str, shapes: Dict[str, tuple]) -> ModelConfig:
  specs: List[LayerSpec] = []
  carried: Dict[str, int] = {}
  for i, entry in enumerate(raw["layers"]):
    kind = entry["type"]
    if kind not in TYPES:
      raise ValueError(f"layer {i}: unknown mixer {kind!r}")
    mixer, fixed = TYPES[kind]
    params = {**copy.deepcopy(entry["mixer"]), **fixed, "layer": i}
    j = params.get("kv_from")
    if j is not None:
      source = specs[j] if 0 <= j < i else None
      if source is None or source.mixer != mixer or source.params.get("kv_from") is not None:
        raise ValueError(f"layer {i}: layer {j} has no keys and values to read")
      if any(source.params[n] != params[n] for n in ("kv_heads", "dim", "vdim")):
        raise ValueError(f"layer {i}: heads differ from those of layer {j}, whose keys and values it reads")
      source.params["lent"] = True
      carried[f"kv{j}"] = RotaryAttention.lent_width(params)
    specs.append(LayerSpec(mixer, params, **_feed_forward(i, entry.get("mlp"))))
  moes = [s.moe for s in specs if s.moe is not None]
  experts = max((m["expert"]["ff"] for m in moes), default=0)
  return ModelConfig(
    model_id=model_id, model_type="tapupel", vocab_size=raw["vocab"], dim=raw["width"], n_layers=len(specs),
    norm_eps=float(raw["norm"]["eps"]), max_seq_len=max_positions(raw), layer_specs=specs,
    embed_scale=float(raw["embedding"]["scale"]), carried=carried,
    n_experts=max((m["router"]["experts"] for m in moes), default=0), moe_intermediate_dim=experts,
    intermediate_dim=max([experts, *(s.ff for s in specs)]),
    torch_dtype=_DTYPE_MAP.get(raw.get("torch_dtype", "bfloat16"), torch.bfloat16),
    bos_token_id=raw.get("bos_token_id"), eos_token_id=raw.get("eos_token_id"),
  )


class TapupelLayer(nn.Module):
  def __init__(self, cfg: ModelConfig, spec: LayerSpec):
    super().__init__()
    self.eps = cfg.norm_eps
    self.mix = MIXERS[spec.mixer](cfg.dim, spec.params, cfg.norm_eps)
    self.mlp = DenseMLP(cfg, spec.ff) if spec.ff else GroupedExperts(cfg.dim, spec.moe) if spec.moe is not None else None
    norms = ("norm1", "norm2") if self.mlp is not None else ("norm1",)
    for n in norms:
      self.register_parameter(n, nn.Parameter(torch.zeros(cfg.dim)))
    self.init_ranges = {n: (-0.2, 0.2) for n in norms}

  def step(self, x, h, cache, rows, after):
    y = self.mix(h, cache, rows)
    x, h = mo.sandwich_norm(y, x, self.norm1, mo.STREAM if self.mlp is not None else after, self.eps)
    if self.mlp is not None:
      x, h = mo.sandwich_norm(self.mlp(h), x, self.norm2, after, self.eps)
    return x, h

  def key_map(self, src: str, dst: str) -> Dict[str, str]:
    m = self.mix.key_map(src + "mix.", dst + "mix.")
    m[src + "norm1"] = dst + "norm1"
    if self.mlp is not None:
      m[src + "norm2"] = dst + "norm2"
    if isinstance(self.mlp, GroupedExperts):
      m.update(self.mlp.key_map(src + "mlp.", dst + "mlp."))
    elif self.mlp is not None:
      m[src + "mlp.gate"] = dst + "mlp.gate_up_proj.weight#0"
      m[src + "mlp.up"] = dst + "mlp.gate_up_proj.weight#1"
      m[src + "mlp.down"] = dst + "mlp.down_proj.weight"
    return m


class TapupelModel(LayeredModel):
  def make_layer(self, cfg: ModelConfig, spec: LayerSpec, place: int) -> nn.Module:
    return TapupelLayer(cfg, spec)

  @staticmethod
  def entry(layer, cache=None):
    return mo.STREAM


def key_map_tapupel(shard: Shard, cfg: ModelConfig) -> Dict[str, str]:
  return layered_key_map(TapupelModel, shard, cfg)
