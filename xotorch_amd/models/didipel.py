"""Sharded Didipel decoder: layers listed one by one in the configuration.

Each layer has a mixer of the kind its entry names (models/mixers.py: window
attention and a gated delta rule side by side, or RWKV-style time mixing), a
dense SwiGLU feed-forward or none, and norms before AND after each sublayer
with weights stored around zero. The residual stream is fp32 throughout (also
between ring stages, `hidden_dtype`); sublayers read and write the model's
dtype, and one fused kernel adds a sublayer's normed output to the stream and
norms the stream for the next sublayer.

Same forward contract as ShardedModel, with one addition: the model is
`slot_indexed`. A step may name the state slot of each of its rows and how
many tokens each row brings, so a batch can be any set of slots and prompts
of unequal length. State per slot is constant in the sequence length (a ring
of one attention window, recurrent matrices, a few last inputs); no zeroing
is needed between requests, position 0 starts from nothing.
"""
from __future__ import annotations

import copy
import os
from typing import Dict, List, Optional

import torch
import torch.nn as nn

from xotorch_amd.models.config import _DTYPE_MAP, LayerSpec, ModelConfig
from xotorch_amd.models.llama import MLP, XotLinear
from xotorch_amd.models.mixers import MIXERS, WindowBiasAttention
from xotorch_amd.ops import mixer_ops as mo
from xotorch_amd.shard import Shard

# nothing in the design bounds positions; this bounds what a request may ask for
DEFAULT_MAX_SEQ = 1 << 20


def didipel_config(raw: dict, model_id: str, shapes: Dict[str, tuple]) -> ModelConfig:
  """config.json (and, for sizes it leaves open, the tensor shapes)."""
  specs: List[LayerSpec] = []
  for i, entry in enumerate(raw["layers"]):
    kind = entry["type"]
    if kind not in MIXERS:
      raise ValueError(f"layer {i}: unknown mixer {kind!r}")
    mlp = entry.get("mlp")
    if mlp is not None and mlp["kind"] != "dense":
      raise ValueError(f"layer {i}: unknown feed-forward {mlp['kind']!r}")
    params = copy.deepcopy(entry["mixer"])
    params["width"] = raw["width"]
    MIXERS[kind].fill_sizes(params, shapes, f"l{i}.mix.")
    specs.append(LayerSpec(kind, params, mlp["ff"] if mlp is not None else 0))
  max_seq = int(raw.get("max_position_embeddings", DEFAULT_MAX_SEQ))
  if os.getenv("XOT_MAX_SEQ_LEN"):
    max_seq = min(max_seq, int(os.environ["XOT_MAX_SEQ_LEN"]))
  return ModelConfig(
    model_id=model_id, model_type="didipel", vocab_size=raw["vocab"], dim=raw["width"], n_layers=len(specs),
    norm_eps=float(raw["norm"]["eps"]), max_seq_len=max_seq, layer_specs=specs,
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


class DidipelLayer(nn.Module):
  def __init__(self, cfg: ModelConfig, spec: LayerSpec):
    super().__init__()
    norms = ("norm1", "norm1b") + (("norm2", "norm2b") if spec.ff else ())
    for n in norms:
      self.register_parameter(n, nn.Parameter(torch.zeros(cfg.dim)))
    self.init_ranges = {n: (-0.2, 0.2) for n in norms}
    self.mix = MIXERS[spec.mixer](cfg.dim, spec.params, cfg.norm_eps)
    self.mlp = DenseMLP(cfg, spec.ff) if spec.ff else None


class DidipelModel(nn.Module):
  """Layer range [shard.start_layer .. shard.end_layer] of a Didipel model."""

  slot_indexed = True
  hidden_dtype = torch.float32

  def __init__(self, cfg: ModelConfig, shard: Shard):
    super().__init__()
    self.cfg, self.shard = cfg, shard
    if shard.is_first_layer:
      self.embed_tokens = nn.Embedding(cfg.vocab_size, cfg.dim)
    self.layers = nn.ModuleDict({str(i): DidipelLayer(cfg, cfg.layer_specs[i])
                                 for i in range(shard.start_layer, shard.end_layer + 1)})
    self.init_ranges = {}
    if shard.is_last_layer:
      self.norm = nn.Parameter(torch.zeros(cfg.dim))
      self.init_ranges["norm"] = (-0.2, 0.2)
      self.lm_head = XotLinear(cfg.dim, cfg.vocab_size, bias=False)

  def reset_rope(self):
    """Position tables (here: distance buckets) after meta construction."""
    device = next(self.parameters()).device
    for m in self.modules():
      if isinstance(m, WindowBiasAttention):
        m.reset_tables(device)

  @property
  def local_layer_ids(self) -> List[int]:
    return list(range(self.shard.start_layer, self.shard.end_layer + 1))

  def pack_decode_weights(self, reserve_bytes: int = 8 << 30) -> int:
    """Same prepack policy as ShardedModel."""
    from xotorch_amd.models.llama import ShardedModel
    return ShardedModel.pack_decode_weights(self, reserve_bytes)

  def head_weight(self):
    return self.lm_head.weight

  def forward(self, x, caches, positions, start_pos: int, is_decode: bool = False, seq_lens=None,
              last_only: bool = True, slots: Optional[torch.Tensor] = None, lens: Optional[torch.Tensor] = None,
              layers_out: Optional[list] = None):
    """x: [B,S] tokens or [B,S,D] fp32 stream. A decode step takes each row's
    position from `positions` ([1] or [B]); a prefill chunk starts at
    `start_pos` in every row, row b bringing lens[b] tokens (None: S). slots:
    int32 [B], the state slot of each row (None: row b is slot b; -1: parked).
    layers_out collects the stream after every local layer."""
    dtype = self.layers[str(self.shard.start_layer)].norm1.dtype
    eps = self.cfg.norm_eps
    B, S = x.shape[0], x.shape[1]
    rows = mo.StepRows(is_decode, 0 if is_decode else int(start_pos),
                       positions.reshape(-1) if is_decode else None, slots, lens)
    if x.dtype in (torch.int32, torch.int64):
      x = self.embed_tokens(x).float()
    elif not (torch.is_grad_enabled() and x.requires_grad):
      x = x.float().clone()  # updated in place below; the caller keeps its own
    layers = [self.layers[str(i)] for i in self.local_layer_ids]
    h = mo.prenorm(x, layers[0].norm1, eps, dtype)
    whole = is_decode or not last_only or S == 1  # the head reads every row
    for i, layer in enumerate(layers):
      if i + 1 < len(layers):
        after = layers[i + 1].norm1
      else:
        after = self.norm if self.shard.is_last_layer and whole else None
      y = layer.mix(h, caches[i] if caches is not None else None, rows)
      x, h = mo.sandwich_norm(y, x, layer.norm1b, layer.norm2 if layer.mlp is not None else after, eps)
      if layer.mlp is not None:
        x, h = mo.sandwich_norm(layer.mlp(h), x, layer.norm2b, after, eps)
      if layers_out is not None:
        layers_out.append(x.clone())
    if not self.shard.is_last_layer:
      return x
    if not whole:
      if lens is None:
        x = x[:, -1:].contiguous()
      else:
        x = x[torch.arange(B, device=x.device), lens.long() - 1][:, None].contiguous()
      h = mo.prenorm(x, self.norm, eps, dtype)
    logits = self.lm_head(h)
    return logits[:, -1] if is_decode or last_only else logits


def key_map_didipel(shard: Shard, cfg: ModelConfig) -> Dict[str, str]:
  """Checkpoint tensor names → DidipelModel parameters."""
  with torch.device("meta"):
    model = DidipelModel(cfg, shard)  # the mixers know where their parts lie
  m: Dict[str, str] = {}
  if shard.is_first_layer:
    m["embed"] = "embed_tokens.weight"
  for lid in model.local_layer_ids:
    src, dst, layer = f"l{lid}.", f"layers.{lid}.", model.layers[str(lid)]
    m.update(layer.mix.key_map(src + "mix.", dst + "mix."))
    m[src + "norm1"], m[src + "norm1b"] = dst + "norm1", dst + "norm1b"
    if layer.mlp is not None:
      m[src + "norm2"], m[src + "norm2b"] = dst + "norm2", dst + "norm2b"
      m[src + "mlp.gate"] = dst + "mlp.gate_up_proj.weight#0"
      m[src + "mlp.up"] = dst + "mlp.gate_up_proj.weight#1"
      m[src + "mlp.down"] = dst + "mlp.down_proj.weight"
  if shard.is_last_layer:
    m["final.norm"], m["head"] = "norm", "lm_head.weight"
  return m
