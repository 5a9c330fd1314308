"""Weight loading: shard-aware HF safetensors → ShardedModel, plus random init.

Parity with the reference's loader (/root/reference/xotorch/inference/torch/llm_utils.py:230-333)
minus the q/k permute (our RoPE uses the HF rotate-half convention, so HF
tensors load verbatim). Only files containing this shard's layers are read —
the same weight_map-driven selection the downloader uses for its
allow-patterns (/root/reference/xotorch/download/new_shard_download.py:181-194).
"""
from __future__ import annotations

import json
from pathlib import Path
from typing import Dict, Optional

import torch

from xotorch_amd.models.config import ModelConfig
from xotorch_amd.models.llama import ShardedModel, hf_key_map as _hf_key_map_llama
from xotorch_amd.shard import Shard


def hf_key_map(shard, cfg):
  """Checkpoint key map, routed by architecture."""
  mtype = getattr(cfg, "model_type", "llama")
  if mtype == "gemma2":
    from xotorch_amd.models.gemma2 import hf_key_map_gemma2
    return hf_key_map_gemma2(shard, cfg)
  if mtype in ("deepseek_v3", "deepseek_v2"):
    from xotorch_amd.models.deepseek_v3 import hf_key_map_deepseek
    return hf_key_map_deepseek(shard, cfg)
  if mtype == "didipel":
    from xotorch_amd.models.didipel import key_map_didipel
    return key_map_didipel(shard, cfg)
  if mtype == "lebotar":
    from xotorch_amd.models.lebotar import key_map_lebotar
    return key_map_lebotar(shard, cfg)
  if mtype == "tapupel":
    from xotorch_amd.models.tapupel import key_map_tapupel
    return key_map_tapupel(shard, cfg)
  if mtype == "dupolorn":
    from xotorch_amd.models.dupolorn import key_map_dupolorn
    return key_map_dupolorn(shard, cfg)
  return _hf_key_map_llama(shard, cfg)


def shard_file_set(model_dir: Path, shard: Shard, cfg: ModelConfig) -> Optional[Dict[str, list]]:
  """Map safetensors filename → [hf keys this shard needs from it]."""
  index_path = model_dir / "model.safetensors.index.json"
  mapping = hf_key_map(shard, cfg)
  if not index_path.exists():
    single = model_dir / "model.safetensors"
    if single.exists():
      return {single.name: list(mapping.keys())}
    return None
  with open(index_path) as f:
    weight_map: Dict[str, str] = json.load(f)["weight_map"]
  files: Dict[str, list] = {}
  for hf_key in mapping:
    fn = weight_map.get(hf_key)
    if fn is not None:
      files.setdefault(fn, []).append(hf_key)
  return files


def load_shard_weights(model: ShardedModel, model_dir: Path, device: str = "cpu") -> int:
  """Load this shard's tensors from HF safetensors files. Returns #tensors."""
  from safetensors import safe_open

  model_dir = Path(model_dir)
  cfg, shard = model.cfg, model.shard
  mapping = hf_key_map(shard, cfg)
  files = shard_file_set(model_dir, shard, cfg)
  if files is None:
    raise FileNotFoundError(f"no safetensors found under {model_dir}")
  tensors: Dict[str, torch.Tensor] = {}
  for fn, keys in files.items():
    with safe_open(str(model_dir / fn), framework="pt", device=device) as f:
      names = set(f.keys())
      for hf_key in keys:
        if hf_key in names:
          tensors[hf_key] = f.get_tensor(hf_key)
  placed_missing = [k for k, our in mapping.items() if "@" in our and k not in tensors]
  if placed_missing:
    raise RuntimeError(f"missing weights for shard {shard}: {placed_missing[:8]}")
  state = remap_hf_state(tensors, mapping, {n: p.shape for n, p in model.named_parameters()})
  missing, unexpected = model.load_state_dict(state, strict=False)
  # tied-embedding models ship no lm_head tensor; rope buffers are computed
  real_missing = [m for m in missing if not m.startswith("rope_")]
  if cfg.tie_word_embeddings:
    real_missing = [m for m in real_missing if m != "lm_head.weight"]
  if real_missing:
    raise RuntimeError(f"missing weights for shard {shard}: {real_missing[:8]}")
  if cfg.tie_word_embeddings and hasattr(model, "lm_head") and not hasattr(model, "embed_tokens"):
    # last shard of a tied model without the embedding: need the embed tensor
    if "lm_head.weight" not in state:
      raise RuntimeError("tied-embedding model: last shard requires model.embed_tokens.weight")
  return len(state)


def remap_hf_state(sd: Dict[str, torch.Tensor], mapping: Dict[str, str],
                   shapes: Optional[Dict[str, tuple]] = None) -> Dict[str, torch.Tensor]:
  """Apply an hf_key_map to an in-memory HF state dict (shared by the
  safetensors path, tests and converters). Three forms of target:
  `key` renames; `key#N` parts are concatenated along dim 0 in N order;
  `key@row` / `key@row,col` parts are placed at an offset of the parameter
  `key`, whose shape comes from `shapes`, with zeros where nothing is placed
  (fused projections with aligned or padded parts). `key@row<axis,lo:hi` places
  that range of the tensor only; several such targets are joined by `;`."""
  state: Dict[str, torch.Tensor] = {}
  packed: Dict[str, Dict[int, torch.Tensor]] = {}
  for hf_key, our in mapping.items():
    if hf_key not in sd:
      continue
    if "#" in our:
      base, part = our.split("#")
      packed.setdefault(base, {})[int(part)] = sd[hf_key]
    elif "@" in our:
      for target in our.split(";"):
        target, _, part = target.partition("<")
        base, offset = target.split("@")
        t = sd[hf_key]
        if part:
          axis, lo, hi = (int(v) for v in part.replace(":", ",").split(","))
          t = t.narrow(axis, lo, hi - lo)
        if base not in state:
          state[base] = torch.zeros(shapes[base], dtype=t.dtype, device=t.device)
        t = t.reshape((1,) * (state[base].dim() - t.dim()) + tuple(t.shape))
        at = [int(o) for o in offset.split(",")]
        at += [0] * (t.dim() - len(at))
        if any(o + n > m for o, n, m in zip(at, t.shape, state[base].shape)):
          raise RuntimeError(f"{hf_key} {tuple(t.shape)} does not fit {base} {tuple(state[base].shape)} at {at}")
        state[base][tuple(slice(o, o + n) for o, n in zip(at, t.shape))] = t
    else:
      state[our] = sd[hf_key]
  for base, parts in packed.items():
    state[base] = torch.cat([parts[i] for i in sorted(parts)], dim=0)
  return state


def _init_ranges(model) -> Dict[str, tuple]:
  """Parameters that only make sense in a range of their own (decays, mixing
  weights, norms of mixers): modules list them in `init_ranges`."""
  return {f"{mod}.{p}" if mod else p: r for mod, m in model.named_modules()
          for p, r in getattr(m, "init_ranges", {}).items()}


def _zero_padding(model):
  """Modules whose parameters are padded keep zeros there."""
  for m in model.modules():
    if hasattr(m, "zero_padding"):
      m.zero_padding()


@torch.no_grad()
def random_init(model: ShardedModel, seed: int = 1234, std: float = 0.02) -> None:
  """Deterministic random init (synthetic-weights benches and tests).

  Per-parameter generator seeding keyed by the parameter NAME so a split
  model and a full model get identical layer weights (the split-vs-full
  logits-equality oracle depends on this).
  """
  import zlib
  ranges = _init_ranges(model)
  for name, p in model.named_parameters():
    # a tied-embedding last shard without the embedding holds a COPY of the
    # embedding matrix as its head: seed it as the embedding so split == full
    seed_name = name
    if name == "lm_head.weight" and model.cfg.tie_word_embeddings:
      seed_name = "embed_tokens.weight"
    g = torch.Generator(device="cpu")
    # stable across processes (python's str hash is salted per process)
    g.manual_seed((seed + zlib.crc32(seed_name.encode())) % (2**63))
    cpu_t = torch.empty(p.shape, dtype=torch.float32)
    if name.endswith("layernorm.weight") or name.endswith("norm.weight"):
      cpu_t.fill_(1.0)
    elif name in ranges:
      cpu_t.uniform_(*ranges[name], generator=g)
    elif name.endswith(".bias"):
      cpu_t.zero_()
    else:
      cpu_t.normal_(0.0, std, generator=g)
    p.copy_(cpu_t.to(device=p.device, dtype=p.dtype))
  _zero_padding(model)


@torch.no_grad()
def fast_random_init_gpu(model: ShardedModel, seed: int = 1234, std: float = 0.02) -> None:
  """GPU-side random init for huge models (70B+): not split-equal across
  shard boundaries, but orders of magnitude faster — weight VALUES don't
  affect decode throughput, only shapes do."""
  g = torch.Generator(device="cuda")
  g.manual_seed(seed)
  ranges = _init_ranges(model)
  for name, p in model.named_parameters():
    if name.endswith("norm.weight"):
      p.fill_(1.0)
    elif name in ranges:
      p.copy_(torch.empty(p.shape, dtype=torch.float32, device=p.device).uniform_(*ranges[name], generator=g))
    elif name.endswith(".bias"):
      p.zero_()
    else:
      tmp = torch.empty(p.shape, dtype=torch.float32, device=p.device)
      tmp.normal_(0.0, std, generator=g)
      p.copy_(tmp.to(p.dtype))
      del tmp
  _zero_padding(model)
