"""Dupolorn decoder (models/layered.py): latent attention, with or without a
sink and an output gate, and matrix memories; a dense feed-forward, a sparse one
whose weights multiply the experts' input, or none. Mixer and feed-forward read
the same stream side by side, through norms with one number each; the mixer's
input passes a short causal convolution. What a layer hands on is an average of
the stream after the embedding and after every layer so far, made by the kernel
that adds the sublayers' outputs and norms the result for the next layer. Token
pairs have embeddings of their own.
"""
from __future__ import annotations

import copy
from typing import Dict, List

import torch
import torch.nn as nn

from xotorch_amd.models.config import _DTYPE_MAP, LayerSpec, ModelConfig
from xotorch_amd.models.didipel import DenseGeluMLP
from xotorch_amd.models.experts import GroupedExperts
from xotorch_amd.models.layered import LayeredModel, layered_key_map, max_positions
from xotorch_amd.models.mixers import MIXERS
from xotorch_amd.ops import mixer_ops as mo
from xotorch_amd.shard import Shard

# layer type in config.json -> mixer, and what the design fixes about it
TYPES = {
  "latent_attention": ("latent_attention", {}),
  "latent_attention_2": ("latent_attention", {"sink": True, "gate": True}),
  "mlstm": ("mlstm", {}),
}


def _feed_forward(i: int, mlp) -> dict:
  if mlp is None:
    return {}
  if mlp["kind"] == "dense":
    return {"ff": mlp["ff"]}
  if mlp["kind"] != "moe":
    raise ValueError(f"layer {i}: unknown feed-forward {mlp['kind']!r}")
  shared = mlp.get("shared")
  return {"moe": {"expert": {"ff": mlp["expert"]["ff"], "act": "relu2"},
                  "shared": {"ff": shared["ff"], "gated": False} if shared else None,
                  "router": {"experts": mlp["router"]["experts"], "top": mlp["router"]["top"], "weights": "sigmoid",
                             "corrected": False, "applied": "input"}}}


def dupolorn_config(raw: dict, model_id: str, shapes: Dict[str, tuple]) -> ModelConfig:
  specs: List[LayerSpec] = []
  for i, entry in enumerate(raw["layers"]):
    kind = entry["type"]
    if kind not in TYPES:
      raise ValueError(f"layer {i}: unknown mixer {kind!r}")
    mixer, fixed = TYPES[kind]
    specs.append(LayerSpec(mixer, {**copy.deepcopy(entry["mixer"]), **fixed}, **_feed_forward(i, entry.get("mlp")),
                           conv=int(raw["canon"]["taps"])))
    if specs[-1].conv < 1:
      raise ValueError(f"input convolution of {specs[-1].conv} taps")
  bigram = {n: int(raw["embedding"]["bigram"][n]) for n in ("buckets", "mul_prev", "mul_cur")}
  if bigram["buckets"] < 1:
    raise ValueError(f"{bigram['buckets']} rows for token pairs")
  moes = [s.moe for s in specs if s.moe is not None]
  experts = max((m["expert"]["ff"] for m in moes), default=0)
  return ModelConfig(
    model_id=model_id, model_type="dupolorn", vocab_size=raw["vocab"], dim=raw["width"], n_layers=len(specs),
    norm_eps=float(raw["norm"]["eps"]), max_seq_len=max_positions(raw), layer_specs=specs,
    embed_scale=float(raw["embedding"]["scale"]), bigram=bigram, final_logit_softcapping=float(raw.get("logit_softcap") or 0.0),
    carried={"streams": len(specs) * raw["width"]},
    n_experts=max((m["router"]["experts"] for m in moes), default=0), moe_intermediate_dim=experts,
    intermediate_dim=max([experts, *(s.ff for s in specs)]),
    torch_dtype=_DTYPE_MAP.get(raw.get("torch_dtype", "bfloat16"), torch.bfloat16),
    bos_token_id=raw.get("bos_token_id"), eos_token_id=raw.get("eos_token_id"),
  )


class DupolornLayer(nn.Module):
  def __init__(self, cfg: ModelConfig, spec: LayerSpec, place: int):
    super().__init__()
    self.eps = cfg.norm_eps
    self.mix = MIXERS[spec.mixer](cfg.dim, spec.params, cfg.norm_eps)
    self.mlp = DenseGeluMLP(cfg, spec.ff) if spec.ff else GroupedExperts(cfg.dim, spec.moe) if spec.moe is not None else None
    norms = ("norm1", "norm2") if self.mlp is not None else ("norm1",)
    for n in norms:
      self.register_parameter(n, nn.Parameter(torch.ones(())))
    self.taps = nn.Parameter(torch.zeros(cfg.dim, spec.conv))
    self.average = nn.Parameter(torch.zeros(place + 2))  # of the embedding and of every layer up to this one
    self.init_ranges = {**{n: (0.8, 1.2) for n in norms}, "taps": (-0.3, 0.3), "average": (0.1, 0.5)}

  def reads(self, cache) -> mo.Reads:
    # the convolution's inputs follow the mixer's state
    ring = cache[len(self.mix.branches)][0] if cache is not None else None
    return mo.Reads((self.norm1,) if self.mlp is None else (self.norm1, self.norm2), self.taps, ring)

  def step(self, x, h, cache, rows, after):
    if self.mlp is None:
      y, z = self.mix(h[0], cache, rows), None
    else:
      y, z = mo.side_by_side(lambda: self.mix(h[0], cache, rows), lambda: self.mlp(h[1]))
    head = isinstance(after, nn.Parameter)
    x, h = mo.depth_norm(y, z, x, self.average, mo.Reads((after,)) if head else after, self.eps, y.dtype, rows)
    return x, h[0] if head else h

  def key_map(self, src: str, dst: str) -> Dict[str, str]:
    m = self.mix.key_map(src + "mix.", dst + "mix.")
    m[src + "norm1"], m[src + "canon1"], m[src + "dwa"] = dst + "norm1", dst + "taps", dst + "average"
    if self.mlp is not None:
      m[src + "norm2"] = dst + "norm2"
    if isinstance(self.mlp, GroupedExperts):
      m.update(self.mlp.key_map(src + "mlp.", dst + "mlp."))
    elif self.mlp is not None:
      m[src + "mlp.gate"] = dst + "mlp.gate_up_proj.weight#0"
      m[src + "mlp.up"] = dst + "mlp.gate_up_proj.weight#1"
      m[src + "mlp.down"] = dst + "mlp.down_proj.weight"
    return m


class DupolornModel(LayeredModel):
  hip = ("_hip_ops", "_hip_stream", "_hip_scan")

  def __init__(self, cfg: ModelConfig, shard: Shard):
    super().__init__(cfg, shard)
    if shard.is_first_layer:
      self.embed_pairs = nn.Embedding(cfg.bigram["buckets"] + 1, cfg.dim)

  def make_layer(self, cfg: ModelConfig, spec: LayerSpec, place: int) -> nn.Module:
    return DupolornLayer(cfg, spec, place)

  def make_final_norm(self):
    self.norm = nn.Parameter(torch.ones(()))
    self.init_ranges["norm"] = (0.8, 1.2)

  @staticmethod
  def entry(layer, cache=None):
    return layer.reads(cache)

  def read(self, x, what, rows, dtype):
    if isinstance(what, mo.Reads):
      return mo.read_stream(x, what, self.cfg.norm_eps, dtype, rows)
    return mo.read_stream(x, mo.Reads((what,)), self.cfg.norm_eps, dtype, rows)[0]

  def embed(self, tokens, caches, rows):
    last = caches[0][-1][0] if caches is not None else None
    rows.depth = mo.Depth(self.embed_tokens.weight, tokens.shape, 1 + len(self.local_layer_ids),
                          keep=rows.streamed)
    return mo.embed_pairs(tokens, self.embed_tokens.weight, self.cfg.embed_scale, self.embed_pairs.weight,
                          self.cfg.bigram, last, rows)

  def receive(self, x, rows, dtype):
    D = self.cfg.dim
    now, *streams = x.float().split(D, dim=-1)
    rows.depth = mo.Depth(x, x.shape[:-1], self.shard.end_layer + 2, D, keep=rows.streamed)
    for t in streams[:self.shard.start_layer + 1]:
      rows.depth.add(t)
    return now.contiguous()

  def hand_on(self, x, rows):
    """The stream and all it has been, still in fp32."""
    short = len(self.cfg.layer_specs) - len(rows.depth.streams)
    return torch.cat([x, *rows.depth.streams, x.new_zeros(*x.shape[:-1], short * self.cfg.dim)], dim=-1)


def key_map_dupolorn(shard: Shard, cfg: ModelConfig) -> Dict[str, str]:
  m = layered_key_map(DupolornModel, shard, cfg)
  if shard.is_first_layer:
    m["bigram"] = "embed_pairs.weight"
  return m
