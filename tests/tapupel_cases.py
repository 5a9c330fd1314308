"""Small random Tapupel checkpoints for the tests."""
import copy

import torch

MOE = {"kind": "moe", "expert": {"ff": 40}, "router": {"experts": 7, "top": 3}}
SHARED = {**MOE, "shared": {"ff": 100}}  # wider than an expert
DENSE = {"kind": "dense", "ff": 88}
DIFF = {"heads": 4, "kv_heads": 2, "dim": 20, "vdim": 12, "diff": 0.3, "scale": 0.31, "rot": {"base": 500.0, "dims": 12}}
BASE = {
  "architecture": "Tapupel", "vocab": 101, "width": 72, "norm": {"eps": 1e-5}, "embedding": {"scale": 1.7},
  "layers": [
    {"type": "rglru", "mlp": SHARED, "mixer": {"width": 96, "blocks": 4, "conv": 4}},
    {"type": "attention_2", "mlp": DENSE, "mixer": DIFF},
    {"type": "attention", "mlp": None, "mixer": {
      "heads": 6, "kv_heads": 2, "dim": 24, "vdim": 24, "scale": 0.2, "softcap": 4.0, "mask": {"size": 11, "keep_first": 3},
      "rot": {"base": 300.0, "dims": 16, "scaling": {"factor": 4.0, "low": 1.0, "high": 3.0, "original": 48}}}},
    {"type": "attention_2", "mlp": MOE, "mixer": {**DIFF, "scale": 0.4, "diff": 0.6, "kv_from": 1}},
    {"type": "attention", "mlp": SHARED, "mixer": {
      "heads": 4, "kv_heads": 4, "dim": 32, "vdim": 32, "scale": 0.18, "softcap": 9.0, "mask": {"size": 33, "keep_first": 1},
      "rot": {"base": 900.0, "dims": 32, "scaling": {"factor": 2.0, "low": 2.0, "high": 5.0, "original": 100}}}},
    {"type": "attention_2", "mlp": None, "mixer": {
      "heads": 3, "kv_heads": 1, "dim": 16, "vdim": 40, "diff": 0.1, "scale": 0.25, "rot": {"base": 100.0, "dims": 2}}},
    {"type": "rglru", "mlp": DENSE, "mixer": {"width": 70, "blocks": 7, "conv": 2}},
    {"type": "attention_2", "mlp": SHARED, "mixer": {**DIFF, "kv_from": 1}},
  ],
}


def small(**changes):
  cfg = copy.deepcopy(BASE)
  cfg.update(copy.deepcopy(changes))
  return cfg


def random_weights(cfg, seed=0, settled=False):
  """Weights at sizes where every mechanism moves the logits: decays spread
  over (0, 1), queries and keys that make softmaxes uneven, caps that bite.
  settled: the stream's first channel is a constant that no sublayer touches
  and that chooses every layer's experts. All rounded to bfloat16, as a
  checkpoint holds them."""
  g = torch.Generator().manual_seed(seed)
  w = {}

  def normal(name, *shape, std=None):
    w[name] = torch.randn(*shape, generator=g) * (shape[-1] ** -0.5 if std is None else std)

  def uniform(name, lo, hi, *shape):
    w[name] = torch.rand(*shape, generator=g) * (hi - lo) + lo

  D = cfg["width"]

  def mlp(p, ff):
    normal(p + "gate", ff, D, std=1.5 * D ** -0.5)
    normal(p + "up", ff, D, std=1.5 * D ** -0.5)
    normal(p + "down", D, ff)

  normal("embed", cfg["vocab"], D, std=1.0)
  if settled:
    w["embed"][:, 0] = 2.0
  for i, layer in enumerate(cfg["layers"]):
    p, m = f"l{i}.mix.", layer["mixer"]
    for n in ("norm1",) + (("norm2",) if layer["mlp"] else ()):
      normal(f"l{i}.{n}", D, std=0.3)
      if settled:
        w[f"l{i}.{n}"][0] = -1.0
    if layer["type"] == "rglru":
      W, n = m["width"], m["width"] // m["blocks"]
      for b in ("y", "x"):
        normal(p + b, W, D)
        normal(f"{p}{b}.b", W, std=0.5)
      normal(p + "conv", W, m["conv"], std=0.6)
      normal(p + "conv.b", W, std=0.3)
      for gate in ("ra", "ri"):
        normal(p + gate, m["blocks"], n, n, std=1.2 * n ** -0.5)
        normal(f"{p}{gate}.b", m["blocks"], n, std=0.7)
      uniform(p + "lam", -7.0, 0.5, W)
      normal(p + "o", D, W)
    else:
      H, G, d, e = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
      maps = 2 if layer["type"] == "attention_2" else 1
      normal(p + "q", H * maps * d, D)
      if maps == 2:
        uniform(p + "q.norm", 0.5, 1.8, d)
        for n in ("lq1", "lk1", "lq2", "lk2"):
          normal(p + n, d, std=0.25)
      if m.get("kv_from") is None:
        normal(p + "k", G * maps * d, D)
        if maps == 2:
          uniform(p + "k.norm", 0.5, 1.8, d)
          normal(p + "v", G * e, D)
      normal(p + "o", D, H * e)
    p, m = f"l{i}.mlp.", layer["mlp"]
    if m is None:
      continue
    if m["kind"] == "dense":
      mlp(p, m["ff"])
      continue
    E = m["router"]["experts"]
    normal(p + "router", E, D, std=(0.1 if settled else 1.0) * D ** -0.5)
    if settled:
      w[p + "router"][:, 0] = 0.4 * torch.randperm(E, generator=g)
    for e in range(E):
      mlp(f"{p}e{e}.", m["expert"]["ff"])
    if m.get("shared"):
      mlp(p + "shared.", m["shared"]["ff"])
      normal(p + "shared.sg", 1, D)
  normal("final.norm", D, std=0.3)
  normal("head", cfg["vocab"], D)
  return {n: t.to(torch.bfloat16) for n, t in w.items()}
