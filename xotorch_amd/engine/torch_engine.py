"""The PyTorch-ROCm engine: our ShardedModel + HIP ops + device-resident KV.

Engine parity with the reference's torchtune engine
(/root/reference/xotorch/inference/torch/sharded_inference_engine.py:37-424),
redesigned MI355X-first:
- hidden states stay bf16 on-device between calls (the numpy fp32 round trip
  exists only at the legacy Node/NumPy boundary for multi-host transport);
- KV caches + position state are engine-owned and never serialized
  (the reference ships mask/tokens/input_pos as JSON per hop);
- all GPU work is serialized through a 1-thread executor (same concurrency
  model as the reference, :46), keeping the asyncio API responsive;
- train/evaluate are real (CE loss, backward from a received ring gradient,
  optimizer step) — the reference declares but never implements them.
"""
from __future__ import annotations

import asyncio
import os
from concurrent.futures import ThreadPoolExecutor
from dataclasses import dataclass, field
from pathlib import Path
from typing import Dict, Optional, Tuple

import numpy as np
import torch

from xotorch_amd import ops
from xotorch_amd.engine.interface import InferenceEngine
from xotorch_amd.engine.kvcache import ShardKVCache, make_cache
from xotorch_amd.engine.state import ShardInferenceState
from xotorch_amd.engine.tokenizers import DummyTokenizer, resolve_tokenizer
from xotorch_amd.models import model_class_for
from xotorch_amd.models.config import ModelConfig, config_from_hf
from xotorch_amd.models.llama import ShardedModel
from xotorch_amd.models.registry import builtin_config, get_repo
from xotorch_amd.models.weights import load_shard_weights, random_init
from xotorch_amd.shard import Shard

TEMP = float(os.getenv("XOT_TEMP", "0.6"))
TOP_K = int(os.getenv("XOT_TOP_K", "35"))
DEFAULT_MAX_GEN = int(os.getenv("XOT_MAX_GEN", "512"))


class ContextExhausted(RuntimeError):
  """Generation reached the model context / KV capacity; the request must be
  finished gracefully (the reference crashes past max_seq_len)."""


@dataclass
class Session:
  cache: ShardKVCache
  state: ShardInferenceState = field(default_factory=ShardInferenceState)


class TorchEngine(InferenceEngine):
  def __init__(self, shard_downloader=None, require_hip: bool = False, device: Optional[str] = None,
               dtype: Optional[torch.dtype] = None):
    self.shard_downloader = shard_downloader
    self.require_hip = require_hip
    if device is None:
      device = "cuda" if torch.cuda.is_available() else "cpu"
    self.device = device
    self.dtype = dtype if dtype is not None else (torch.bfloat16 if device == "cuda" else torch.float32)
    self.shard: Optional[Shard] = None
    self.model: Optional[ShardedModel] = None
    self.cfg: Optional[ModelConfig] = None
    self.tokenizer = None
    self.sessions: Dict[str, Session] = {}
    self._executor = ThreadPoolExecutor(max_workers=1)
    self._rng = torch.Generator(device=self.device)
    self._rng.manual_seed(int(os.getenv("XOT_SEED", "1234")))
    self.oom_count = 0

  # ---------- model lifecycle ----------

  async def ensure_shard(self, shard: Shard):
    if self.shard == shard and self.model is not None:
      return
    model_dir: Optional[Path] = None
    if self.shard_downloader is not None:
      try:
        model_dir = await self.shard_downloader.ensure_shard(shard, type(self).__name__)
      except Exception:
        model_dir = None
    await asyncio.get_running_loop().run_in_executor(self._executor, self._build_model, shard, model_dir)
    # tokenizer
    if model_dir is not None and (Path(model_dir) / "tokenizer_config.json").exists():
      self.tokenizer = await resolve_tokenizer(model_dir)
    else:
      repo = get_repo(shard.model_id, type(self).__name__)
      if repo in (None, "dummy") or os.getenv("XOT_OFFLINE", "0") == "1":
        self.tokenizer = DummyTokenizer()
      else:
        try:
          self.tokenizer = await resolve_tokenizer(repo)
        except Exception:
          self.tokenizer = DummyTokenizer()

  def _build_model(self, shard: Shard, model_dir: Optional[Path]):
    cfg_dict = None
    if model_dir is not None and (Path(model_dir) / "config.json").exists():
      cfg_dict = str(Path(model_dir) / "config.json")
    else:
      cfg_dict = builtin_config(shard.model_id)
    if cfg_dict is None:
      raise ValueError(f"no config available for model {shard.model_id}")
    cfg = config_from_hf(cfg_dict, model_id=shard.model_id)
    model_cls = model_class_for(cfg)
    # construct at the target dtype so to_empty materializes it directly
    # (fp32-then-cast would peak at 2x the weight bytes)
    prev_dtype = torch.get_default_dtype()
    torch.set_default_dtype(self.dtype)
    try:
      with torch.device("meta"):
        model = model_cls(cfg, shard)
    finally:
      torch.set_default_dtype(prev_dtype)
    model = model.to_empty(device=self.device)
    model = model.to(self.dtype)
    # recompute rope tables (to_empty leaves buffers uninitialized); each
    # decoder derives its own table shape (MLA uses qk_rope_head_dim)
    model.reset_rope()
    if model_dir is not None and (
      (Path(model_dir) / "model.safetensors.index.json").exists() or (Path(model_dir) / "model.safetensors").exists()
    ):
      load_shard_weights(model, Path(model_dir), device="cpu")
      model = model.to(self.device)
    else:
      random_init(model)
    model.eval()
    if self.device == "cuda":
      # decode-GEMM weight prepack (auto-picked vs hipBLASLt per shape at
      # first decode); keep headroom for per-request KV caches
      torch.cuda.empty_cache()
      model.pack_decode_weights(reserve_bytes=24 << 30)
    self.model = model
    self.cfg = cfg
    self.shard = shard
    self.sessions.clear()

  def _session(self, request_id: str, batch: int, total_len: int) -> Session:
    sess = self.sessions.get(request_id)
    if sess is None or sess.cache.batch != batch or sess.cache.capacity < total_len:
      cache = make_cache(self.cfg, self.shard, batch, total_len, self.dtype, self.device)
      sess = Session(cache=cache, state=ShardInferenceState(total_len=total_len, batch=batch))
      self.sessions[request_id] = sess
    return sess

  async def clear_session(self, request_id: str):
    self.sessions.pop(request_id, None)

  # ---------- tokenizer plumbing ----------

  async def encode(self, shard: Shard, prompt: str) -> np.ndarray:
    await self.ensure_shard(shard)
    tokens = self.tokenizer.encode(prompt)
    return np.asarray(tokens, dtype=np.int64)

  async def decode(self, shard: Shard, tokens) -> str:
    await self.ensure_shard(shard)
    return self.tokenizer.decode(list(np.asarray(tokens).reshape(-1)))

  async def sample(self, x: np.ndarray, temp: float = TEMP, top_k: int = TOP_K,
                   top_p: float = 0.0) -> np.ndarray:
    logits = torch.from_numpy(np.asarray(x))
    if logits.dim() == 3:
      logits = logits[:, -1, :]
    tok = ops.softmax_sample(logits, temperature=temp, top_k=top_k, top_p=top_p)
    return tok.cpu().numpy()

  # ---------- inference ----------

  async def infer_tensor(
    self, request_id: str, shard: Shard, input_data: np.ndarray, inference_state: Optional[dict] = None
  ) -> Tuple[np.ndarray, Optional[dict]]:
    await self.ensure_shard(shard)
    loop = asyncio.get_running_loop()
    return await loop.run_in_executor(self._executor, self._infer_tensor_sync, request_id, input_data, inference_state)

  def _infer_tensor_sync(self, request_id: str, input_data: np.ndarray, inference_state: Optional[dict]):
    meta = ShardInferenceState.from_dict(inference_state)
    x = torch.from_numpy(np.ascontiguousarray(input_data))
    if (inference_state or {}).get("wire_dtype") == "bfloat16" and x.dtype == torch.int16:
      # bf16 hidden state shipped as raw int16 bytes (numpy has no bf16)
      x = x.view(torch.bfloat16)
    is_tokens = x.dtype in (torch.int32, torch.int64)
    B = x.shape[0]
    S = x.shape[1]
    total_len = meta.total_len or min(self.cfg.max_seq_len, S + DEFAULT_MAX_GEN)
    sess = self._session(request_id, B, total_len)
    # Each stage tracks its OWN position: every stage of the ring processes
    # the same chunks in the same order, so the local counter is always the
    # chunk's start. (Position state never travels.)
    start_pos = sess.state.curr_pos
    if start_pos + S > min(self.cfg.max_seq_len, sess.cache.capacity):
      raise ContextExhausted(
        f"request {request_id}: position {start_pos + S} exceeds context "
        f"(max_seq_len {self.cfg.max_seq_len}, cache capacity {sess.cache.capacity})"
      )
    x = x.to(self.device)
    if not is_tokens:
      x = x.to(getattr(self.model, "hidden_dtype", self.dtype))
    positions = torch.arange(start_pos, start_pos + S, dtype=torch.int32, device=self.device)
    is_decode = S == 1 and start_pos > 0
    try:
      with torch.inference_mode():
        out = self.model(
          x, caches=sess.cache.caches, positions=positions, start_pos=start_pos, is_decode=is_decode,
        )
    except torch.cuda.OutOfMemoryError:
      self.oom_count += 1
      self.sessions.pop(request_id, None)
      if self.device == "cuda":
        torch.cuda.empty_cache()
      raise
    new_pos = start_pos + S
    sess.state.curr_pos = new_pos
    sess.state.total_len = total_len
    # merge pass-through metadata (max_tokens, traceparent, ...) so request
    # attributes survive the hop — engines own only their position keys
    out_state = dict(inference_state or {})
    out_state.update({"curr_pos": new_pos, "total_len": total_len, "batch": B})
    if not self.shard.is_last_layer and out.dtype == torch.bfloat16:
      # mid-ring hidden states travel as bf16 bytes (half the wire bytes of
      # the reference's fp32-numpy hop); last-stage logits stay fp32 for the
      # local sampling site
      out_np = out.contiguous().cpu().view(torch.int16).numpy()
      out_state["wire_dtype"] = "bfloat16"
    else:
      out_np = out.float().cpu().numpy()
      out_state.pop("wire_dtype", None)
    return out_np, out_state

  # ---------- training (capability the reference declared but never built) ----------

  async def train(self, request_id: str, shard: Shard, inputs, targets, lengths, loss: str = "ce", opt=None):
    await self.ensure_shard(shard)
    loop = asyncio.get_running_loop()
    return await loop.run_in_executor(
      self._executor, self._train_sync, request_id, inputs, targets, lengths, loss, opt, True
    )

  async def evaluate(self, request_id: str, shard: Shard, inputs, targets, lengths, loss: str = "ce"):
    await self.ensure_shard(shard)
    loop = asyncio.get_running_loop()
    return await loop.run_in_executor(
      self._executor, self._train_sync, request_id, inputs, targets, lengths, loss, None, False
    )

  def _train_forward(self, x: torch.Tensor):
    """Training/eval forward THROUGH THE MODEL's own cache-free path
    (caches=None): one forward implementation for inference and training —
    drift between them is impossible by construction.
    Activation checkpointing inside the model is opt-in
    (XOT_ACT_CKPT=1): measured 380 vs 283 ms/step on 8B LoRA B=8 — worth it
    only when activations would not fit."""
    S = x.shape[1]
    positions = torch.arange(0, S, dtype=torch.int32, device=self.device)
    return self.model(x, caches=None, positions=positions, start_pos=0, last_only=False)

  _lora_applied = False

  def _maybe_apply_lora(self):
    """XOT_LORA_RANK>0 switches training to LoRA adapters (lazy, once)."""
    rank = int(os.getenv("XOT_LORA_RANK", "0"))
    if rank > 0 and not self._lora_applied:
      from xotorch_amd.train.lora import apply_lora
      apply_lora(self.model, rank=rank, alpha=float(os.getenv("XOT_LORA_ALPHA", str(2 * rank))))
      self._lora_applied = True
      self._opt = None  # rebuild over the adapter params

  def _ce_loss(self, out, tgt, lengths):
    lens = torch.from_numpy(np.ascontiguousarray(lengths)).to(self.device)
    S = tgt.shape[1]
    mask = torch.arange(S, device=self.device)[None, :] < lens[:, None]
    lg = out.float().reshape(-1, out.shape[-1])
    lt = tgt.reshape(-1).long()
    ce = torch.nn.functional.cross_entropy(lg, lt, reduction="none").reshape(tgt.shape)
    return (ce * mask).sum() / mask.sum().clamp(min=1)

  def _train_sync(self, request_id, inputs, targets, lengths, loss, opt, do_step):
    self._maybe_apply_lora()
    model = self.model
    was_training = model.training
    model.train(do_step)
    x = torch.from_numpy(np.ascontiguousarray(inputs)).to(self.device)
    is_tokens = x.dtype in (torch.int32, torch.int64)
    if not do_step and loss != "back_gradient":
      # evaluation: loss only, under no_grad — a backward here would leave
      # accumulated grads contaminating the next optimizer step
      if not model.shard.is_last_layer:
        raise ValueError("non-last shard evaluates by forwarding activations, not locally")
      with torch.no_grad():
        out = self._train_forward(x)
        tgt = torch.from_numpy(np.ascontiguousarray(targets)).to(self.device)
        loss_val = float(self._ce_loss(out, tgt, lengths))
      model.train(was_training)
      return loss_val, None
    if not is_tokens:
      x = x.to(getattr(model, "hidden_dtype", self.dtype)).requires_grad_(True)
    with torch.enable_grad():
      out = self._train_forward(x)
      if loss == "back_gradient":
        # backward from the gradient received off the ring (targets = dL/d(out))
        grad = torch.from_numpy(np.ascontiguousarray(targets)).to(self.device).to(out.dtype)
        out.backward(grad)
        loss_val = 0.0
      else:
        tgt = torch.from_numpy(np.ascontiguousarray(targets)).to(self.device)
        if model.shard.is_last_layer:
          loss_t = self._ce_loss(out, tgt, lengths)
          loss_t.backward()
          loss_val = float(loss_t.detach())
        else:
          raise ValueError("non-last shard must train with loss='back_gradient'")
    if do_step:
      if opt is None:
        opt = self._default_optimizer()
      opt.step()
      opt.zero_grad(set_to_none=True)
    in_grad = None
    if not is_tokens and x.grad is not None:
      in_grad = x.grad.float().cpu().numpy()
    model.train(was_training)
    return loss_val, in_grad

  _opt = None

  def _default_optimizer(self):
    if self._opt is None:
      params = [p for p in self.model.parameters() if p.requires_grad]
      self._opt = torch.optim.AdamW(params, lr=float(os.getenv("XOT_LR", "1e-5")))
    return self._opt

  # ---------- checkpointing ----------

  async def save_checkpoint(self, shard: Shard, path: str):
    await self.ensure_shard(shard)
    from safetensors.torch import save_file
    Path(path).parent.mkdir(parents=True, exist_ok=True)
    if self._lora_applied:
      from xotorch_amd.train.lora import lora_state_dict
      sd = {k: v.contiguous() for k, v in lora_state_dict(self.model).items()}
    else:
      sd = {k: v.detach().contiguous().cpu() for k, v in self.model.state_dict().items() if not k.startswith("rope_")}
    save_file(sd, path)

  async def load_checkpoint(self, shard: Shard, path: str):
    await self.ensure_shard(shard)
    from safetensors import safe_open
    with safe_open(path, framework="pt", device="cpu") as f:
      sd = {k: f.get_tensor(k) for k in f.keys()}
    self.model.load_state_dict(sd, strict=False)
