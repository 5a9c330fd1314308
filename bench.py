#!/usr/bin/env python3
"""Driver benchmark: ring-pipeline decode tokens/sec (whole ring) + p50 TTFT.

Measures BASELINE.json's headline metric — Llama-3-70B sharded across N GPUs
of one node as ring pipeline stages (RCCL send/recv over xGMI), greedy decode
on synthetic prompts with random-init weights (no network for datasets or
checkpoints).

Launch (driver contract):
  python bench.py --gpus 1 --steps K --warmup W                 # single GPU
  python -m torch.distributed.run --nnodes=1 --nproc-per-node N \
      --master-addr 127.0.0.1 bench.py --gpus N --steps K --warmup W

One "step" advances every in-flight micro-batch by one token; value =
whole-job decode tokens/sec = global_batch * steps / elapsed (max over ranks).
Scaling is weak: micro-batch count = N pipeline stages with fixed per-mb
batch, so per-GPU work (its layer shard's weight stream per step) is constant
as N grows.
"""
import argparse
import json
import os
import statistics
import sys
import time
from pathlib import Path

sys.path.insert(0, str(Path(__file__).resolve().parent))

# hipBLASLt/rocBLAS algorithm selection pre-tuned on MI355X (gfx950) for the
# bench GEMM shapes; read-only (tuning off) so TTFT stays clean. Must be set
# before torch initializes.
_tuned = Path(__file__).resolve().parent / "profiles" / "tunableop_gfx950.csv"
if _tuned.exists() and os.getenv("XOT_TUNABLEOP", "1") == "1":
  # TunableOp inserts the device ordinal before ".csv" when resolving the
  # filename -- stage per-ordinal copies it will actually find.
  import shutil
  base = Path("/tmp/xot_tunableop.csv")
  for i in list(range(8)) + [""]:
    dst = Path(f"/tmp/xot_tunableop{i}.csv")
    if not dst.exists():
      shutil.copyfile(_tuned, dst)
  os.environ.setdefault("PYTORCH_TUNABLEOP_ENABLED", "1")
  os.environ.setdefault("PYTORCH_TUNABLEOP_TUNING", "0")
  os.environ.setdefault("PYTORCH_TUNABLEOP_FILENAME", str(base))

import torch  # noqa: E402


def _gemma2_like(width, n_layers, ff, vocab, kv_heads, window):
  return {
    "model_type": "gemma2", "hidden_size": width, "num_hidden_layers": n_layers,
    "num_attention_heads": width // 128, "num_key_value_heads": kv_heads, "head_dim": 128,
    "intermediate_size": ff, "vocab_size": vocab, "rms_norm_eps": 1e-6, "max_position_embeddings": 1 << 20,
    "tie_word_embeddings": True, "query_pre_attn_scalar": 128, "attn_logit_softcapping": 50.0,
    "final_logit_softcapping": 30.0, "sliding_window": window,
  }


def _didipel_pair(model_id):
  """The registry's Didipel of that size, and gemma2 (sandwich norms, sliding
  windows) with the same width, depth, heads, feed-forward, vocabulary."""
  from xotorch_amd.models.registry import builtin_config
  cfg = builtin_config(model_id)
  left = next(e["mixer"]["left"] for e in cfg["layers"] if e["type"] == "parallel")
  like = _gemma2_like(cfg["width"], len(cfg["layers"]), cfg["layers"][0]["mlp"]["ff"], cfg["vocab"],
                      left["kv_heads"], left["mask"]["size"])
  return [(model_id, cfg), ("gemma2 of that size", like)]


def _lebotar_pair(model_id):
  """The registry's Lebotar of that size, and deepseek (latent attention and
  group-limited sigmoid routing in every layer) with the same width, depth,
  heads, latent, experts, vocabulary. It always has a shared expert besides."""
  from xotorch_amd.models.registry import builtin_config
  cfg = builtin_config(model_id)
  moe = cfg["layers"][0]["mlp"]
  lat = next(e["mixer"] for e in cfg["layers"] if e["type"] == "latent_attention")
  like = {
    "model_type": "deepseek_v3", "hidden_size": cfg["width"], "num_hidden_layers": len(cfg["layers"]),
    "num_attention_heads": lat["heads"], "num_key_value_heads": lat["heads"],
    "intermediate_size": moe["expert"]["ff"], "moe_intermediate_size": moe["expert"]["ff"],
    "n_routed_experts": moe["router"]["experts"], "num_experts_per_tok": moe["router"]["top"], "n_shared_experts": 1,
    "n_group": moe["router"]["groups"]["count"], "topk_group": moe["router"]["groups"]["keep"],
    "routed_scaling_factor": moe["router"]["scale"], "norm_topk_prob": False, "first_k_dense_replace": 0,
    "q_lora_rank": 0, "kv_lora_rank": lat["kv_rank"], "qk_rope_head_dim": lat["rot_dim"],
    "qk_nope_head_dim": lat["dim"], "v_head_dim": lat["vdim"], "vocab_size": cfg["vocab"],
    "rope_theta": 10000.0, "rms_norm_eps": 1e-6, "max_position_embeddings": 8192,
  }
  return [(model_id, cfg), ("deepseek of that size", like)]


def _tapupel_pair(model_id):
  """The registry's Tapupel of that size, and lebotar (local attention, latent
  attention, selective scan, sparse feed-forwards) with the same width, depth,
  heads, experts, vocabulary. It has no shared experts."""
  from xotorch_amd.models.registry import builtin_config
  cfg = builtin_config(model_id)
  att = next(e["mixer"] for e in cfg["layers"] if e["type"] == "attention")
  moe = cfg["layers"][0]["mlp"]
  width, dim = cfg["width"], att["dim"]
  like = {
    "attention": ("attention", {"heads": att["heads"], "kv_heads": att["kv_heads"], "dim": dim, "vdim": dim,
                                "scale": dim ** -0.5, "v_mix": False, "mask": {"size": att["mask"]["size"]}}),
    "attention_2": ("latent_attention", {"heads": att["heads"], "dim": dim, "rot_dim": dim // 2, "vdim": dim,
                                         "kv_rank": 4 * dim, "rot": {"base": 10000.0, "dims": dim // 2},
                                         "scale": (dim + dim // 2) ** -0.5}),
    "rglru": ("mamba1", {"inner": 2 * width, "state": 16, "conv": 4, "dt_rank": width // 16}),
  }
  mlp = {"kind": "moe", "expert": {"ff": moe["expert"]["ff"], "limit": 7.0},
         "router": {**moe["router"], "scale": 2.5, "groups": {"count": 8, "keep": 4}}}
  return [(model_id, cfg), ("lebotar of that size", {
    "architecture": "Lebotar", "vocab": cfg["vocab"], "width": width, "norm": cfg["norm"], "residual_mult": 0.5,
    "layers": [{"type": like[e["type"]][0], "mixer": like[e["type"]][1], "mlp": mlp} for e in cfg["layers"]]})]


def _dupolorn_pair(model_id):
  """The registry's Dupolorn of that size, and lebotar (latent attention,
  selective scan, sigmoid routing) with the same width, depth, heads, latent,
  experts, vocabulary. Its experts have two products before the activation and
  two thirds of the width, and it chooses one more in place of the shared one."""
  from xotorch_amd.models.registry import builtin_config
  cfg = builtin_config(model_id)
  width, moe = cfg["width"], cfg["layers"][0]["mlp"]
  lat = next(e["mixer"] for e in cfg["layers"] if e["type"] == "latent_attention")
  like = {"latent_attention": ("latent_attention", lat), "latent_attention_2": ("latent_attention", lat),
          "mlstm": ("mamba1", {"inner": 2 * width, "state": 16, "conv": 4, "dt_rank": width // 16})}
  mlp = {"kind": "moe", "expert": {"ff": moe["expert"]["ff"] * 2 // 3, "limit": 7.0},
         "router": {"experts": moe["router"]["experts"], "top": moe["router"]["top"] + 1, "scale": 2.5,
                    "groups": {"count": 8, "keep": 4}}}
  return [(model_id, cfg), ("lebotar of that size", {
    "architecture": "Lebotar", "vocab": cfg["vocab"], "width": width, "norm": cfg["norm"], "residual_mult": 0.5,
    "layers": [{"type": like[e["type"]][0], "mixer": like[e["type"]][1], "mlp": mlp} for e in cfg["layers"]]})]


DESIGNS = {"didipel": _didipel_pair, "lebotar": _lebotar_pair, "tapupel": _tapupel_pair, "dupolorn": _dupolorn_pair}


def design_bench(args):
  """One JSON line per (model, batch x prompt): prompt and decode tokens/s on
  one GPU, random weights. The pair takes turns at every shape."""
  from xotorch_amd.parallel.comm import init_distributed
  from xotorch_amd.parallel.ring import RingPipeline
  init_distributed()
  device = args.device or ("cuda" if torch.cuda.is_available() else "cpu")

  def sync():
    if device == "cuda":
      torch.cuda.synchronize()

  from xotorch_amd.models.registry import BUILTIN_CONFIGS
  prefix = f"{args.design}-"
  sizes = args.sizes or ",".join(m[len(prefix):] for m in BUILTIN_CONFIGS if m.startswith(prefix) and not m.endswith("-dummy"))
  for size in sizes.split(","):
    for shape in args.shapes.split(","):
      batch, prompt = (int(v) for v in shape.split("x"))
      for name, cfg in DESIGNS[args.design](f"{args.design}-{size}"):
        ring = RingPipeline(name, 0, 1, device, torch.bfloat16 if args.dtype == "bf16" else torch.float32,
                            mb_batch=batch, prompt_len=prompt, max_gen=args.warmup + args.steps + 4,
                            use_graphs=not args.no_graphs, cfg_override=cfg)
        ring.prefill()  # first calls: library heuristics, allocator
        ring.use_graphs = False  # captured; only the prompts run again
        ms = min(ring.prefill().ttft_ms[0] for _ in range(3))
        for _ in range(args.warmup):
          ring.decode_step()
        sync()
        t0 = time.perf_counter()
        for _ in range(args.steps):
          ring.decode_step()
        sync()
        step = (time.perf_counter() - t0) / args.steps
        print(json.dumps({
          "model": name, "size": size, "batch": batch, "prompt": prompt, "dtype": args.dtype,
          "params_b": round(sum(p.numel() for p in ring.model.parameters()) / 1e9, 3),
          "state_mib": round(ring.caches[0].nbytes() / 2**20, 1),
          "prefill_tokens_per_s": round(batch * prompt / ms * 1e3), "prefill_ms": round(ms, 2),
          "decode_tokens_per_s": round(batch / step), "decode_ms_per_step": round(step * 1e3, 3),
        }), flush=True)
        del ring
        if device == "cuda":
          torch.cuda.empty_cache()


def main():
  p = argparse.ArgumentParser()
  p.add_argument("--gpus", type=int, default=1)
  p.add_argument("--steps", type=int, default=32)
  p.add_argument("--warmup", type=int, default=8)
  p.add_argument("--model", type=str, default="llama-3-70b")
  p.add_argument("--mb-batch", type=int, default=128, help="sequences per micro-batch (per pipeline slot)")
  p.add_argument("--prompt-len", type=int, default=512)
  p.add_argument("--no-graphs", action="store_true")
  p.add_argument("--device", type=str, default=None)
  p.add_argument("--dtype", type=str, default="bf16", choices=["bf16", "fp32"])
  p.add_argument("--design", choices=sorted(DESIGNS), default=None,
                 help="instead: prefill and decode throughput of a design beside the closest other model at equal size")
  p.add_argument("--sizes", type=str, default=None, help="with --design: sizes to run (default: all of the registry)")
  p.add_argument("--shapes", type=str, default="1x4096,32x1024,128x512",
                 help="with --design: batch x prompt tokens, comma separated")
  args = p.parse_args()
  if args.design:
    return design_bench(args)

  from xotorch_amd.parallel.comm import init_distributed, max_over_ranks
  import torch.distributed as dist

  rank, world = init_distributed()
  if world != args.gpus and int(os.getenv("WORLD_SIZE", "1")) != args.gpus:
    # --gpus describes the intended N; trust the actual world size
    pass
  device = args.device or ("cuda" if torch.cuda.is_available() else "cpu")
  dtype = torch.bfloat16 if args.dtype == "bf16" else torch.float32
  cfg_override = None
  if device == "cpu" and args.model == "llama-3-70b":
    # CPU smoke path (no GPU in dev container): tiny model, same code path;
    # give it >= world layers so every rank gets a shard
    from xotorch_amd.models.registry import builtin_config
    args.model = "dummy"
    args.prompt_len = min(args.prompt_len, 128)  # dummy max_seq_len is 256
    world_hint = int(os.getenv("WORLD_SIZE", "1"))
    if world_hint > 4:
      cfg_override = dict(builtin_config("dummy"))
      cfg_override["num_hidden_layers"] = world_hint

  from xotorch_amd.parallel.ring import RingPipeline

  max_gen = args.warmup + args.steps + 4
  ring = RingPipeline(
    model_id=args.model, rank=rank, world=world, device=device, dtype=dtype,
    mb_batch=args.mb_batch, prompt_len=args.prompt_len, max_gen=max_gen,
    use_graphs=not args.no_graphs, cfg_override=cfg_override,
  )
  global_batch = args.mb_batch * ring.M

  # ---- prefill (TTFT measured at the last stage) ----
  stats = ring.prefill()
  ttfts = torch.tensor(stats.ttft_ms, dtype=torch.float64, device="cpu")
  if world > 1:
    # TTFT lives on the last stage; ship it to rank 0 (gloo groups move it
    # on host, nccl on device)
    if device == "cuda" and dist.get_backend() != "gloo":
      ttfts = ttfts.to(device)
    dist.broadcast(ttfts, world - 1)
    ttfts = ttfts.cpu()
  p50_ttft = float(statistics.median(ttfts.tolist()))

  # ---- warmup ----
  for _ in range(args.warmup):
    ring.decode_step()

  # ---- timed region ----
  if device == "cuda":
    torch.cuda.synchronize()
  if dist.is_initialized():
    dist.barrier()
  if device == "cuda":
    torch.cuda.synchronize()
  t0 = time.perf_counter()
  for _ in range(args.steps):
    ring.decode_step()
  if device == "cuda":
    torch.cuda.synchronize()
  if dist.is_initialized():
    dist.barrier()
  if device == "cuda":
    torch.cuda.synchronize()
  elapsed = time.perf_counter() - t0
  elapsed = max_over_ranks(elapsed, device if device == "cuda" else "cpu")
  ring.finish()

  tokens = global_batch * args.steps
  toks_per_s = tokens / elapsed
  ms_per_step = elapsed / args.steps * 1000.0

  if rank == 0:
    result = {
      "metric": "decode tokens/sec (whole ring)",
      "value": round(toks_per_s, 2),
      "unit": "tokens/s",
      "n_gpus": world,
      "steps": args.steps,
      "warmup": args.warmup,
      "ms_per_step": round(ms_per_step, 3),
      "higher_is_better": True,
      "scaling": "weak",
      "vs_baseline": None,
      "dtype": (args.dtype
                + ("+fp8-w8a8" if os.getenv("XOT_FP8_GEMM", "0") == "1" else "")
                + ("+fp8-kv" if os.getenv("XOT_FP8_KV", "0") == "1" else "")),
      "data": "synthetic",
      "config": {
        "model": args.model,
        "global_batch": global_batch,
        "seq_len": args.prompt_len,
        "parallelism": f"pp{world}",
        "micro_batches": ring.M,
        "mb_batch": args.mb_batch,
        "p50_ttft_ms": round(p50_ttft, 1),
        "ttft_semantics": "whole-batch pipelined prefill (request-level TTFT: serve path)",
        "sampling": "greedy",
        "hip_graphs": not args.no_graphs and device == "cuda",
      },
    }
    print(json.dumps(result))
  if dist.is_initialized():
    dist.destroy_process_group()


if __name__ == "__main__":
  main()
