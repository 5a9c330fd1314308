"""Small random Dupolorn checkpoints for the tests."""
import copy

import torch

MOE = {"kind": "moe", "expert": {"ff": 40}, "router": {"experts": 7, "top": 3}, "shared": {"ff": 100}}  # wider than an expert
ONE = {"kind": "moe", "expert": {"ff": 70}, "router": {"experts": 5, "top": 1}, "shared": {"ff": 24}}
DENSE = {"kind": "dense", "ff": 88}
LATENT = {"heads": 3, "dim": 20, "rot_dim": 12, "vdim": 28, "kv_rank": 44, "scale": 0.3, "rot": {"base": 500.0, "dims": 12}}
GATED = {"heads": 6, "dim": 24, "rot_dim": 8, "vdim": 16, "kv_rank": 56, "scale": 0.25, "rot": {"base": 300.0, "dims": 8}}
MEMORY = {"heads": 5, "dim": 20, "vdim": 36, "gate_cap": 7.0}
BASE = {
  "architecture": "Dupolorn", "vocab": 101, "width": 72, "norm": {"eps": 1e-5}, "logit_softcap": 6.0, "canon": {"taps": 3},
  "embedding": {"scale": 1.7, "bigram": {"buckets": 53, "mul_prev": 7, "mul_cur": 11}},
  "layers": [
    {"type": "mlstm", "mlp": MOE, "mixer": MEMORY},
    {"type": "latent_attention_2", "mlp": ONE, "mixer": GATED},
    {"type": "latent_attention", "mlp": DENSE, "mixer": LATENT},
    {"type": "mlstm", "mlp": None, "mixer": {"heads": 2, "dim": 48, "vdim": 24, "gate_cap": 3.0}},
    {"type": "latent_attention_2", "mlp": DENSE, "mixer": {**GATED, "heads": 17, "dim": 16}},
    {"type": "latent_attention", "mlp": MOE, "mixer": LATENT},
  ],
}


def small(**changes):
  cfg = copy.deepcopy(BASE)
  cfg.update(copy.deepcopy(changes))
  return cfg


def random_weights(cfg, seed=0, settled=False):
  """Weights at sizes where every mechanism moves the logits: memories of a few
  tokens and of many, input gates on either side of zero, queries and keys that
  make softmaxes uneven, sinks among the scores, averages that weigh every depth.
  settled: the stream's first channel is a constant that no sublayer touches and
  that chooses every layer's experts. All rounded to bfloat16, as a checkpoint
  holds them."""
  g = torch.Generator().manual_seed(seed)
  w = {}

  def normal(name, *shape, std=None):
    w[name] = torch.randn(*shape, generator=g) * (shape[-1] ** -0.5 if std is None else std)

  def uniform(name, lo, hi, *shape):
    w[name] = torch.rand(shape, generator=g) * (hi - lo) + lo

  def out(name, *shape):
    normal(name, *shape)
    if settled:
      w[name][0] = 0.0

  D = cfg["width"]
  normal("embed", cfg["vocab"], D, std=1.0)
  normal("bigram", cfg["embedding"]["bigram"]["buckets"] + 1, D, std=1.0)
  if settled:
    w["embed"][:, 0], w["bigram"][:, 0] = 2.0, 0.0
  for i, layer in enumerate(cfg["layers"]):
    p, m = f"l{i}.mix.", layer["mixer"]
    for n in ("norm1",) + (("norm2",) if layer["mlp"] else ()):
      uniform(f"l{i}.{n}", 0.6, 1.5)
    normal(f"l{i}.canon1", D, cfg["canon"]["taps"], std=0.4)
    uniform(f"l{i}.dwa", 0.2, 0.6, i + 2)
    if layer["type"] == "mlstm":
      H, d, e = m["heads"], m["dim"], m["vdim"]
      for n, rows in (("q", H * d), ("k", H * d), ("v", H * e), ("g", H * e), ("i", H), ("f", H)):
        normal(p + n, rows, D)
      normal(p + "i.b", H, std=1.5)
      uniform(p + "f.b", 0.0, 5.0, H)
      uniform(p + "norm", 0.5, 1.8, H * e)
    else:
      H, d, r, e, R = (m[n] for n in ("heads", "dim", "rot_dim", "vdim", "kv_rank"))
      normal(p + "q", H * (d + r), D, std=1.6 * D ** -0.5)
      normal(p + "dkv", R + r, D)
      uniform(p + "dkv.norm", 0.5, 1.8, R)
      normal(p + "uk", H * d, R)
      normal(p + "uv", H * e, R)
      if layer["type"] == "latent_attention_2":
        uniform(p + "sink", 0.0, 5.0, H)
        normal(p + "g", H * e, D)
    out(p + "o", D, m["heads"] * m["vdim"])
    p, m = f"l{i}.mlp.", layer["mlp"]
    if m is None:
      continue
    if m["kind"] == "dense":
      normal(p + "gate", m["ff"], D, std=1.5 * D ** -0.5)
      normal(p + "up", m["ff"], D, std=1.5 * D ** -0.5)
      out(p + "down", D, m["ff"])
      continue
    E = m["router"]["experts"]
    normal(p + "router", E, D, std=(0.1 if settled else 1.0) * D ** -0.5)
    if settled:
      w[p + "router"][:, 0] = 0.4 * torch.randperm(E, generator=g)
    for name, ff in [(f"e{e}.", m["expert"]["ff"]) for e in range(E)] + ([("shared.", m["shared"]["ff"])] if m.get("shared") else []):
      normal(p + name + "up", ff, D, std=1.5 * D ** -0.5)
      out(p + name + "down", D, ff)
  uniform("final.norm", 0.6, 1.5)
  normal("head", cfg["vocab"], D, std=3 * D ** -0.5)
  return {n: t.to(torch.bfloat16) for n, t in w.items()}
