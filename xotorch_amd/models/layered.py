"""Decoders whose layers are listed one by one in the configuration.

ModelConfig.layer_specs names each layer's mixer (models/mixers.py) and its
feed-forward; a design adds its own layer class, which says how norms and the
residual stream surround them. The stream is fp32 throughout (also between
ring stages, `hidden_dtype`); sublayers read and write the model's dtype.

Same forward contract as ShardedModel, with one addition: the model is
`slot_indexed`. A step may name the state slot of each of its rows and how
many tokens each row brings, so a batch can be any set of slots and prompts
of unequal length. No zeroing is needed between requests, position 0 starts
from nothing.
"""
from __future__ import annotations

import os
from typing import Dict, List, Optional

import torch
import torch.nn as nn

from xotorch_amd.models.config import LayerSpec, ModelConfig
from xotorch_amd.models.llama import ShardedModel, XotLinear
from xotorch_amd.ops import mixer_ops as mo
from xotorch_amd.shard import Shard

# nothing in these designs bounds positions; this bounds what a request may ask for
DEFAULT_MAX_SEQ = 1 << 20


def max_positions(raw: dict) -> int:
  n = int(raw.get("max_position_embeddings", DEFAULT_MAX_SEQ))
  env = os.getenv("XOT_MAX_SEQ_LEN")
  return min(n, int(env)) if env else n


class LayeredModel(nn.Module):
  """Layer range [shard.start_layer .. shard.end_layer] of such a model.

  A layer has `norm1`, `mix`, `mlp` or None, `key_map(src, dst)` and `step(x,
  h, cache, rows, after)` -> (stream, what is read next): `after` is the weight
  of the stream's next norm, mo.STREAM for the stream as it is, or None."""

  slot_indexed = True
  hidden_dtype = torch.float32
  hip = ("_hip_ops", "_hip_mixers")

  def make_layer(self, cfg: ModelConfig, spec: LayerSpec, place: int) -> nn.Module:
    raise NotImplementedError

  @staticmethod
  def entry(layer, cache=None):
    """What a layer reads: the stream normed with this weight, or mo.STREAM."""
    return layer.norm1

  def embed(self, tokens, caches, rows):
    x = self.embed_tokens(tokens).float()
    return x * self.cfg.embed_scale if self.cfg.embed_scale != 1.0 else x

  def receive(self, x, rows, dtype):
    """What an earlier ring stage handed on -> the stream."""
    if self.cfg.carried_dim:
      x, *carried = x.split([self.cfg.dim, *self.cfg.carried.values()], dim=-1)
      rows.carried = {name: t.to(dtype) for name, t in zip(self.cfg.carried, carried)}
    if not (torch.is_grad_enabled() and x.requires_grad):
      x = x.float().clone(memory_format=torch.contiguous_format)  # updated in place; the caller keeps its own
    return x

  def hand_on(self, x, rows):
    if not self.cfg.carried_dim:
      return x
    return torch.cat([x, *(rows.carried[name].float() if name in rows.carried else x.new_zeros(*x.shape[:-1], width)
                           for name, width in self.cfg.carried.items())], dim=-1)

  def read(self, x, what, rows, dtype):
    """The stream as a layer or the head reads it."""
    return mo.prenorm(x, what, self.cfg.norm_eps, dtype)

  def extensions(self) -> List[str]:
    """HIP extensions that a forward pass loads (ops/build.py)."""
    return sorted({name for m in self.modules() for name in getattr(m, "hip", ())})

  def __init__(self, cfg: ModelConfig, shard: Shard):
    super().__init__()
    self.cfg, self.shard = cfg, shard
    if shard.is_first_layer:
      self.embed_tokens = nn.Embedding(cfg.vocab_size, cfg.dim)
    self.layers = nn.ModuleDict({str(i): self.make_layer(cfg, spec, i) for i, spec in cfg.shard_specs(shard).items()})
    self.init_ranges = {}
    if shard.is_last_layer:
      self.make_final_norm()
      self.lm_head = XotLinear(cfg.dim, cfg.vocab_size, bias=False)

  def make_final_norm(self):
    self.norm = nn.Parameter(torch.zeros(self.cfg.dim))
    self.init_ranges["norm"] = (-0.2, 0.2)

  def reset_rope(self):
    """Position tables of the mixers after meta construction."""
    device = next(self.parameters()).device
    for m in self.modules():
      if hasattr(m, "reset_tables"):
        m.reset_tables(device)

  @property
  def local_layer_ids(self) -> List[int]:
    return list(range(self.shard.start_layer, self.shard.end_layer + 1))

  def pack_decode_weights(self, reserve_bytes: int = 8 << 30) -> int:
    """Same prepack policy as ShardedModel."""
    return ShardedModel.pack_decode_weights(self, reserve_bytes)

  def head_weight(self):
    return self.lm_head.weight

  def forward(self, x, caches, positions, start_pos: int, is_decode: bool = False, seq_lens=None,
              last_only: bool = True, slots: Optional[torch.Tensor] = None, lens: Optional[torch.Tensor] = None,
              layers_out: Optional[list] = None):
    """x: [B,S] tokens or [B,S,cfg.hidden_dim] fp32 stream (and what travels
    with it). A decode step takes each row's position from `positions` ([1] or
    [B]); a prefill chunk starts at `start_pos` in every row, row b bringing
    lens[b] tokens (None: S). slots: int32 [B], the state slot of each row
    (None: row b is slot b; -1: parked). layers_out collects the stream after
    every local layer."""
    dtype = self.layers[str(self.shard.start_layer)].norm1.dtype
    B, S = x.shape[0], x.shape[1]
    if caches is None and x.is_cuda and not torch.is_grad_enabled():  # the kernels keep state somewhere
      from xotorch_amd.engine.kvcache import make_cache
      caches = make_cache(self.cfg, self.shard, B, S, dtype, x.device).caches
    rows = mo.StepRows(is_decode, 0 if is_decode else int(start_pos),
                       positions.reshape(-1) if is_decode else None, slots, lens, streamed=layers_out is not None)
    if x.dtype in (torch.int32, torch.int64):
      x = self.embed(x, caches, rows)
    else:
      x = self.receive(x, rows, dtype)
    layers = [self.layers[str(i)] for i in self.local_layer_ids]
    states = caches if caches is not None else [None] * len(layers)
    h = self.read(x, self.entry(layers[0], states[0]), rows, dtype)
    whole = is_decode or not last_only or S == 1  # the head reads every row
    for i, layer in enumerate(layers):
      if i + 1 < len(layers):
        after = self.entry(layers[i + 1], states[i + 1])
      else:
        after = self.norm if self.shard.is_last_layer and whole else None
      x, h = layer.step(x, h, states[i], rows, after)
      if layers_out is not None:
        layers_out.append(x.clone())
    if not self.shard.is_last_layer:
      return self.hand_on(x, rows)
    if not whole:
      if lens is None:
        x = x[:, -1:].contiguous()
      else:
        x = x[torch.arange(B, device=x.device), lens.long() - 1][:, None].contiguous()
      h = self.read(x, self.norm, rows, dtype)
    logits = self.lm_head(h)
    if self.cfg.final_logit_softcapping:
      logits = mo.soft_cap(logits, self.cfg.final_logit_softcapping)
    return logits[:, -1] if is_decode or last_only else logits


def layered_key_map(model_cls, shard: Shard, cfg: ModelConfig) -> Dict[str, str]:
  """Checkpoint tensor names → parameters of `model_cls`."""
  with torch.device("meta"):
    model = model_cls(cfg, shard)  # the mixers know where their parts lie
  m: Dict[str, str] = {}
  if shard.is_first_layer:
    m["embed"] = "embed_tokens.weight"
  for lid in model.local_layer_ids:
    m.update(model.layers[str(lid)].key_map(f"l{lid}.", f"layers.{lid}."))
  if shard.is_last_layer:
    m["final.norm"], m["head"] = "norm", "lm_head.weight"
  return m
