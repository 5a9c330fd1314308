"""Trace replay: given token ids through a model, step by step, logits out.

Drives the serving worker (serve_ring.RingSlotWorker, one rank) with a trace
in place of its request queue: prompts go into free slots and prefill in the
scheduler's chunks and batches, single tokens advance their slots in one
decode tick (the captured graph on a GPU). Nothing is sampled.

  trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N

Standard input brings one JSON object a line:

  {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": []}

For every step DIR/<step>.f32 receives the logits at the wanted places (in
the order of the entries and of `want`) as little-endian float32, and a line
`done <step>` is printed. `end` gives the slots of finished requests back.
"""
from __future__ import annotations

import argparse
import json
import sys
from pathlib import Path
from typing import Dict, List, Tuple

import torch

SLOTS = 24


class TraceRunner:
  def __init__(self, worker):
    self.worker = worker
    self.slot: Dict[str, int] = {}
    self.pos: Dict[str, int] = {}

  def _place(self, rid: str) -> int:
    if rid not in self.slot:
      used = set(self.slot.values())
      free = [i for i in range(self.worker.slots) if i not in used]
      if not free:
        raise RuntimeError(f"more than {self.worker.slots} live requests")
      self.slot[rid], self.pos[rid] = free[0], 0
    return self.slot[rid]

  def _prefill(self, entries: List[dict], logits: Dict[Tuple[str, int], torch.Tensor]):
    """Portions of several tokens (or first tokens), chunk by chunk; requests
    that are equally far run as one batch, as in the serving loop."""
    from xotorch_amd import serve_ring
    w = self.worker
    todo = {}
    for e in entries:
      rid, slot, at = e["id"], self._place(e["id"]), self.pos[e["id"]]
      toks = torch.zeros(1, at + len(e["tokens"]), dtype=torch.int64)
      toks[0, at:] = torch.tensor(e["tokens"])
      w._begin_prefill(slot, toks.to(w.device))
      w._pf[slot]["c0"] = at
      todo[slot] = (rid, at, e)
    pending = set(todo)
    while pending:
      c0 = max(w._pf[s]["c0"] for s in pending)
      group = sorted(s for s in pending if w._pf[s]["c0"] == c0)
      if not w.slot_indexed:
        group = group[:1]
      out = w._prefill_hidden(group, c0, last_only=False)
      for row, slot in enumerate(group):
        rid, at, e = todo[slot]
        for place in e["want"]:
          if c0 <= at + place < c0 + serve_ring.PREFILL_CHUNK:
            logits[rid, place] = out[row, at + place - c0].float()
        w._pf[slot]["c0"] = c0 + serve_ring.PREFILL_CHUNK
        if w._pf[slot]["c0"] >= w._pf[slot]["plen"]:
          pending.discard(slot)
          self.pos[rid] = w._pf[slot]["plen"]
          w._activate(slot)

  def _decode(self, entries: List[dict], logits: Dict[Tuple[str, int], torch.Tensor]):
    w = self.worker
    rows = [self.slot[e["id"]] for e in entries]
    w.active = [i in rows for i in range(w.slots)]
    w._reset_inactive()
    at = torch.tensor([self.pos[e["id"]] for e in entries], dtype=torch.int32, device=w.device)
    idx = torch.tensor(rows, dtype=torch.int64, device=w.device)
    w.positions[idx] = at
    w.seq_lens[idx] = at + 1
    w.tok_buf[idx, 0] = torch.tensor([e["tokens"][0] for e in entries], dtype=torch.int64, device=w.device)
    w.run_decode()
    for e, slot in zip(entries, rows):
      self.pos[e["id"]] += 1
      for place in e["want"]:
        logits[e["id"], place] = w.logits_buf[slot].float().clone()

  @torch.inference_mode()
  def step(self, entries: List[dict], end: List[str]) -> torch.Tensor:
    """One step; returns the wanted logits [wanted, vocab]."""
    logits: Dict[Tuple[str, int], torch.Tensor] = {}
    going_on = [e for e in entries if e["id"] in self.slot and len(e["tokens"]) == 1]
    rest = [e for e in entries if e not in going_on]
    if rest:
      self._prefill(rest, logits)
    if going_on:
      self._decode(going_on, logits)
    for rid in end:
      self.worker._release([self.slot.pop(rid)])
      del self.pos[rid]
    rows = [logits[e["id"], place] for e in entries for place in e["want"]]
    return torch.stack(rows).cpu() if rows else torch.empty(0, self.worker.cfg.vocab_size)


def build_extensions(model_dir: str):
  """Compiles what is missing of the HIP extensions that the model runs on."""
  from xotorch_amd.models import config_from_hf, model_class_for
  from xotorch_amd.ops import build as hip_build
  from xotorch_amd.shard import Shard
  cfg = config_from_hf(Path(model_dir) / "config.json", "model")
  with torch.device("meta"):
    model = model_class_for(cfg)(cfg, Shard("model", 0, cfg.n_layers - 1, cfg.n_layers))
  needed = model.extensions() if hasattr(model, "extensions") else ["_hip_ops"]
  hip_build.build(verbose=False, missing_only=True, only=needed)


def build_worker(model_dir: str, dtype: torch.dtype, max_tokens: int):
  from xotorch_amd.serve_ring import RingSlotWorker
  device = "cuda" if torch.cuda.is_available() else "cpu"
  worker = RingSlotWorker(Path(model_dir).name, 0, 1, device=device, dtype=dtype, model_dir=model_dir,
                          slots=SLOTS, max_seq=max_tokens + 2)
  if device == "cuda":
    worker._build_graph()
  return worker


def main(argv=None) -> int:
  p = argparse.ArgumentParser("trace_run", description="replay a trace of token ids, write logits")
  p.add_argument("--model", required=True, help="folder with config.json and model.safetensors")
  p.add_argument("--dtype", choices=["bfloat16", "float32"], default="bfloat16")
  p.add_argument("--out", required=True, help="folder for <step>.f32")
  p.add_argument("--max-tokens", type=int, default=4096, help="most tokens that live requests hold at any time")
  args = p.parse_args(argv)
  if torch.cuda.is_available():
    build_extensions(args.model)
  torch.backends.cuda.matmul.allow_tf32 = False
  runner = TraceRunner(build_worker(args.model, getattr(torch, args.dtype), args.max_tokens))
  for line in sys.stdin:
    if not line.strip():
      continue
    msg = json.loads(line)
    out = runner.step(msg["entries"], msg.get("end", []))
    if out.shape[0]:
      out.numpy().astype("<f4").tofile(str(Path(args.out) / f"{msg['step']}.f32"))
    print(f"done {msg['step']}", flush=True)
  return 0
