"""Tapupel: every mechanism alone, the model through its cache, and serving,
against the plain functions of tapupel_oracle.py. CPU runs take the torch path
in 32-bit, GPU runs the HIP kernels in 32-bit and bfloat16."""
import asyncio
import io
import json

import numpy as np
import pytest
import torch

import tapupel_cases as cases
import tapupel_oracle as oracle
from layered_common import (
  BF16, F32, Session, close, load_model, make_worker, on, on_device, plausible, rnd, rows, run_cut, serve, state_of,
  two_ranks_serve, write_checkpoint,
)
from xotorch_amd.engine.kvcache import make_cache
from xotorch_amd.models.config import config_from_hf
from xotorch_amd.models.experts import GroupedExperts
from xotorch_amd.models.mixers import GatedLinearUnit, RotaryAttention, turn_rates
from xotorch_amd.ops import mixer_ops as mo
from xotorch_amd.shard import Shard

CUTS = ((1, 2, 40, 3, 30), (2,) * 12, (11, 22, 33), (32,), (33, 31, 2), ())
LAST = len(cases.BASE["layers"]) - 1


# ---------------------------------------------------------------- rotation

@pytest.mark.parametrize("dims,base,scaling", [
  (2, 7.0, None), (16, 300.0, None), (16, 300.0, {"factor": 4.0, "low": 1.0, "high": 3.0, "original": 48}),
  (32, 900.0, {"factor": 1.0, "low": 2.0, "high": 5.0, "original": 100}),
  (64, 10000.0, {"factor": 32.0, "low": 1.0, "high": 4.0, "original": 512})])
def test_turn_rates(dims, base, scaling):
  rot = {"base": base, "dims": dims, "scaling": scaling}
  got, want = turn_rates(rot), oracle.frequencies(rot)
  assert len(got) == dims // 2
  np.testing.assert_allclose(got, want, rtol=1e-12)
  if scaling and scaling["factor"] > 1:
    plain = oracle.frequencies({"base": base, "dims": dims})
    ratio = np.array(want) / np.array(plain)
    low = 1 / scaling["factor"]
    # kept, blended and stretched ones all occur
    assert (ratio == 1).any() and np.isclose(ratio, low).any() and ((ratio > low * 1.001) & (ratio < .999)).any()


# ---------------------------------------------------------------- attention

ROT = {"base": 300.0, "scaling": {"factor": 4.0, "low": 1.0, "high": 3.0, "original": 48}}
KEPT = [  # heads, kv_heads, dim, turned dims, window, first tokens kept, cap
  (6, 2, 20, 12, 11, 3, 4.0),
  (4, 4, 64, 64, 33, 1, 9.0),
  (8, 1, 128, 64, 64, 40, 5.0),    # more than a tile of first tokens
  (20, 1, 32, 32, 40, 5, 30.0),    # more query heads on one key head than a tile holds
  (2, 1, 256, 256, 30, 0, 3.0),    # none kept
  (3, 3, 40, 8, 1, 1, 2.0),        # itself and the first
  (2, 2, 80, 2, 1000, 6, 0.0),     # one window, no cap
  (5, 5, 10, 6, 7, 90, 6.0),       # most are kept
]
DIFF = [  # heads, kv_heads, dim, values' dim, turned dims
  (6, 2, 20, 12, 8),
  (4, 4, 64, 128, 64),
  (8, 1, 128, 96, 32),
  (20, 1, 32, 48, 32),
  (4, 1, 128, 256, 128),
  (2, 1, 256, 256, 40),
  (3, 3, 40, 8, 2),
  (2, 2, 18, 20, 18),
]


class Attention:
  """One attention op with its inputs for T tokens; several share a state."""

  def __init__(self, kind, T, H, G, d, e, rot, mask=None, cap=0.0, maps=1, seed=0, diff=.3):
    self.kind, self.T, self.mask, self.maps = kind, T, mask, maps
    self.H, self.G, self.d, self.e, self.rot, self.cap = H, G, d, e, rot, cap
    at_k = 8 + H * maps * d
    self.at = [0, at_k, at_k + 8 + G * maps * d if maps == 2 else at_k]  # parts with gaps
    self.N = self.at[2] + G * max(e, maps * d) + 5
    self.proj = rnd(T, self.N, seed=seed, scale=1.5)
    self.qn, self.kn = ((rnd(d, seed=i) * .2 + 1).to(BF16).double() for i in (1, 2))
    self.scale, self.diff, self.lam, self.source = 1.5 / d ** .5, diff, .43, None

  def heads(self, x, at, n, norm):
    x = x[:, at:at + n * self.maps * self.d].reshape(-1, n, self.maps, self.d)
    if self.maps == 2:
      return oracle.rotate(oracle.rms(x, 1e-5) * norm, self.rot, pairs=True)
    return oracle.rms(oracle.rotate(x, self.rot, pairs=False), 1e-5)

  def inputs(self):
    s = self.source or self
    k = self.heads(s.proj, s.at[1], self.G, s.kn)
    v = s.proj[:, s.at[2]:s.at[2] + self.G * self.e].reshape(-1, self.G, self.e)
    return self.heads(self.proj, self.at[0], self.H, self.qn), k, v

  def expected(self):
    q, k, v = self.inputs()
    if self.maps == 2:
      o = oracle.difference(q, k, v, self.scale, self.lam, self.diff, 1e-5)
    else:
      o = oracle.attention(q[:, :, 0], k[:, :, 0], v, self.scale, self.mask, self.cap or None)
    return .7 * o.reshape(self.T, -1)

  def state(self, slots=3, capacity=512):
    return state_of(RotaryAttention, {"kv_heads": self.G, "dim": self.d, "vdim": self.e, "mask": self.mask,
                                      "diff": self.diff if self.maps == 2 else None}, self.kind, slots, capacity)

  def run(self, x, state, step):
    x, qn, kn = on_device(self.kind, x, self.qn, self.kn)
    mask = self.mask or {"size": 0, "keep_first": 0}
    two, width = self.maps == 2, self.H * self.e
    rule = mo.AttnRule(self.H, self.G, self.d, self.e, self.maps, self.scale, self.cap, mask["size"], mask["keep_first"],
                       two, not two, 1e-5, 1 - self.diff if two else 1.0)
    freq = torch.tensor(oracle.frequencies(self.rot), dtype=F32, device=self.kind[0])
    out = None
    if x.is_cuda:  # columns of a wider tensor
      out = torch.full((*x.shape[:2], (16 + width + 3) // 4 * 4), 9.0, dtype=x.dtype, device=x.device)
    y = mo.rotary_attn(x, self.at[0], (x, self.at[1], self.at[2]), rule, qn if two else None, kn if two else None, freq,
                       torch.tensor([self.lam], dtype=F32, device=self.kind[0]) if two else None, state, step,
                       self.source is None, out=out, out_at=8 if x.is_cuda else 0, out_scale=.7)
    if x.is_cuda:
      assert (y[..., :8] == 9).all() and (y[..., 8 + width:] == 9).all()
      y = y[..., 8:8 + width]
    return y.cpu().double()

  def __call__(self, lo, hi, state, step):
    return self.run(self.proj[None, lo:hi], state, step)[0]


def kept(kind, shape, T, **kw):
  H, G, d, dims, size, keep, cap = shape
  return Attention(kind, T, H, G, d, d, {**ROT, "dims": dims}, {"size": size, "keep_first": keep}, cap, **kw)


def two_maps(kind, shape, T, **kw):
  H, G, d, e, dims = shape
  return Attention(kind, T, H, G, d, e, {"base": 300.0, "dims": dims}, maps=2, **kw)


OPS = [pytest.param(make, shape, id=f"{make.__name__}-{'-'.join(str(v) for v in shape)}")
       for make, shapes in ((kept, KEPT), (two_maps, DIFF)) for shape in shapes]


@on
@pytest.mark.parametrize("make,shape", OPS)
def test_attention_prompt_portions_and_decode(kind, make, shape):
  a = make(kind, shape, 110)
  want = a.expected()
  close(a(0, 110, a.state(), rows(kind)), want, kind[1], 1.5)
  for cuts in CUTS:
    close(run_cut(a, kind, 110, cuts), want, kind[1], 1.5)


def stand_out(a, query, key, map_=0):
  """The key that, of all, the query's map scores highest: equal vectors after
  the turn."""
  v = torch.where(torch.arange(a.d) % 3 == 0, 4.0, -2.0).double()[None]
  span = slice(map_ * a.d, (map_ + 1) * a.d)
  a.proj[query, a.at[0]:a.at[0] + a.H * a.maps * a.d].view(a.H, -1)[:, span] = v
  back = oracle.rotate(v, a.rot, pairs=a.maps == 2, first=query - key).to(BF16).double()
  a.proj[key, a.at[1]:a.at[1] + a.G * a.maps * a.d].view(a.G, -1)[:, span] = back


def last_of(a, kind, query):
  """The query's output in a prompt, right after a cut, two after, and decoded."""
  yield a(0, query + 1, a.state(), rows(kind))[query]
  for cut in (1, 2):
    if query + 1 > cut:
      state, p = a.state(), query + 1 - cut
      a(0, p, state, rows(kind, slots=[1]))
      yield a(p, query + 1, state, rows(kind, start=p, slots=[1]))[-1]
  state = a.state()
  if query:
    a(0, query, state, rows(kind, slots=[1]))
  yield a(query, query + 1, state, rows(kind, True, positions=[query], slots=[1]))[0]


@on
@pytest.mark.parametrize("shape", [(4, 2, 32, 32, 21, 3, 50.0), (2, 2, 128, 64, 64, 33, 50.0), (2, 1, 64, 64, 32, 0, 0.0)])
@pytest.mark.parametrize("past", [-1, 0, 1, 11, 40])  # queries from the window's end on
def test_window_and_first_tokens_show(kind, shape, past):
  """A key that outweighs all others counts if it is in the window or among the
  first ones, and is gone if it is just outside of both."""
  size, keep = shape[4:6]
  query = size + past
  for key in {query - size + 1, query - size, keep - 1, keep, 0, query}:
    if not 0 <= key <= query:
      continue
    a = kept(kind, shape, query + 1)
    a.scale = 40.0 / a.d  # a score of 40
    stand_out(a, query, key)
    want = a.expected()[query]
    alone = .7 * a.inputs()[2][key].repeat_interleave(a.H // a.G, 0).reshape(-1)
    assert ((want - alone).abs().max() < 5e-2) == (query - key < size or key < keep)
    for got in last_of(a, kind, query):
      close(got, want, kind[1])


@on
@pytest.mark.parametrize("query,first,second", [(99, 0, 98), (96, 63, 1), (64, 64, 31), (95, 32, 64), (33, 32, 0), (127, 95, 96)])
def test_far_keys_of_both_maps_show(kind, query, first, second):
  """Each map has its own key that outweighs all others."""
  a = two_maps(kind, (4, 2, 32, 24, 32), query + 1)
  a.scale, a.qn, a.kn = 40.0 / 32, torch.ones(32).double(), torch.ones(32).double()
  stand_out(a, query, first, 0)
  stand_out(a, query, second, 1)
  want = a.expected()[query]
  v = a.inputs()[2]
  alone = .7 * .7 * oracle.rms(v[first] - a.lam * v[second], 1e-5).repeat_interleave(2, 0).reshape(-1)
  assert (want - alone).abs().max() < 5e-2
  for got in last_of(a, kind, query):
    close(got, want, kind[1])


@on
def test_equal_maps_leave_one(kind):
  """With the first map's queries and keys in both, the difference is
  (1 - lambda) times one attention, whose size the norm takes out."""
  a = two_maps(kind, (2, 1, 16, 16, 16), 40)
  for at, n in ((a.at[0], 2), (a.at[1], 1)):
    x = a.proj[:, at:at + n * 32].view(-1, n, 2, 16)
    x[:, :, 1] = x[:, :, 0]
  q, k, v = a.inputs()
  one = oracle.attention(q[:, :, 0], k[:, :, 0], v, a.scale)
  for a.lam in (-.5, 0.0, .25, 1.6):  # past one the sign turns
    want = .7 * .7 * oracle.rms((1 - a.lam) * one, 1e-5).reshape(40, -1)
    close(a(0, 40, a.state(), rows(kind)), want, kind[1])
    close(run_cut(a, kind, 40, (7,)), want, kind[1])


@on
def test_scores_are_capped(kind):
  """Scores far beyond the cap weigh like the cap, and stay finite."""
  a = kept(kind, (2, 1, 32, 2, 64, 0, 1.0), 50)
  a.scale = 30.0
  want = a.expected()
  q, k, v = a.inputs()
  s = (k[:, 0, 0] @ q[49, 0, 0]) * a.scale
  p = torch.softmax(torch.tanh(s), 0)  # nearly two weights only: e and 1 / e
  close(want[49, :32], .7 * (p @ v[:, 0]), F32)
  close(a(0, 50, a.state(), rows(kind)), want, kind[1])
  close(run_cut(a, kind, 50, (20,)), want, kind[1])


@on
@pytest.mark.parametrize("make,shape", [(kept, (6, 2, 64, 32, 21, 4, 8.0)), (two_maps, (6, 2, 40, 24, 20))])
def test_attention_rows_are_independent(kind, make, shape):
  """Unequal lengths in one step, arbitrary slots, a parked row in between,
  ragged decode positions."""
  a, b = make(kind, shape, 90), make(kind, shape, 90, seed=7)
  state = a.state(slots=4)
  for t in state:
    t.fill_(3.0)
  before = [t[0].clone() for t in state]
  got = a.run(torch.stack([a.proj[:70], b.proj[:70], b.proj[:70]]), state, rows(kind, slots=[3, -1, 1], lens=[5, 70, 70]))
  wa, wb = a.expected(), b.expected()
  close(got[0, :5], wa[:5], kind[1])
  assert (got[1] == 0).all() and (got[0, 5:] == 0).all()
  close(got[2], wb[:70], kind[1])
  for i in range(18):
    at = [70 + i, 0, 5 + i]
    got = a.run(torch.stack([op.proj[p:p + 1] for op, p in zip((b, a, a), at)]), state,
                rows(kind, True, positions=at, slots=[1, -1, 3]))
    close(got[0, 0], wb[70 + i], kind[1])
    assert (got[1] == 0).all()
    close(got[2, 0], wa[5 + i], kind[1])
  assert all((t[0] == u).all() for t, u in zip(state, before))


@on
@pytest.mark.parametrize("make,shape", [(kept, (4, 1, 64, 64, 600, 70, 20.0)), (two_maps, (4, 1, 64, 64, 64)), (two_maps, (2, 2, 128, 256, 64))])
def test_long_caches_split_over_blocks(kind, make, shape):
  """Decoding late in a long cache, where several blocks share one row."""
  a = make(kind, shape, 800)
  state = a.state(capacity=1000)
  a(0, 797, state, rows(kind, slots=[2]))
  q, k, v = a.inputs()
  for i in range(797, 800):
    seen = torch.tensor([j for j in range(i + 1) if oracle.sees(i, j, a.mask)])
    want = []
    for h in range(a.H):
      o = []
      for m in range(a.maps):
        s = k[seen, h // (a.H // a.G), m] @ q[i, h, m] * a.scale
        s = a.cap * torch.tanh(s / a.cap) if a.cap else s
        o.append(torch.softmax(s, 0) @ v[seen, h // (a.H // a.G)])
      want.append(o[0] if a.maps == 1 else oracle.rms(o[0] - a.lam * o[1], 1e-5) * (1 - a.diff))
    got = a(i, i + 1, state, rows(kind, True, positions=[i], slots=[2]))[0]
    close(got, .7 * torch.cat(want), kind[1], 1.5)


@on
def test_reading_the_keys_and_values_of_another(kind):
  """A second op has queries, scale and lambda of its own over a first one's
  cache, and writes nothing."""
  a, b = two_maps(kind, (6, 2, 20, 12, 8), 60), two_maps(kind, (6, 2, 20, 12, 8), 60, seed=4, diff=.6)
  b.source, b.scale, b.lam, b.qn = a, .5, -.2, a.qn * .5
  want = b.expected()
  state, got, p = a.state(), [], 0
  for n in (17, 2, 30):
    a(p, p + n, state, rows(kind, start=p, slots=[1]))
    held = [t.clone() for t in state]
    got.append(b(p, p + n, state, rows(kind, start=p, slots=[1])))
    assert all((t == u).all() for t, u in zip(state, held))
    p += n
  for t in range(p, 60):
    step = rows(kind, True, positions=[t], slots=[1])
    a(t, t + 1, state, step)
    got.append(b(t, t + 1, state, step))
  close(torch.cat(got), want, kind[1])


# ---------------------------------------------------------------- gated linear recurrence

UNIT = [  # channels, blocks, taps
  (40, 4, 3), (64, 1, 1), (96, 3, 4), (33, 11, 2), (128, 2, 5), (512, 1, 4), (260, 2, 4), (256, 2, 4), (70, 7, 6), (12, 12, 2)]


class Unit:
  """Convolution, gates, recurrence and gelu branch together."""

  def __init__(self, kind, shape, T, seed=0):
    self.kind, self.T = kind, T
    W, blocks, taps = self.shape = shape
    n = W // blocks
    self.y_at, self.x_at = 4, 4 + (W + 7) // 8 * 8
    self.proj = rnd(T, self.x_at + W + 3, seed=seed)
    self.in_bias, self.conv, self.bias = rnd(2, W, seed=1, scale=.5), rnd(W, taps, seed=2, scale=.6), rnd(W, seed=3, scale=.4)
    self.gates = rnd(2, blocks, n, n, seed=4, scale=1.5 * n ** -.5)
    self.gate_bias = rnd(2, blocks, n, seed=5, scale=.7)
    self.lam = (rnd(W, seed=6, scale=2.0) - 3).to(BF16).double()

  def expected(self):
    W = self.shape[0]
    y = oracle.gelu_tanh(self.proj[:, self.y_at:self.y_at + W] + self.in_bias[0])
    u = oracle.causal_conv(self.proj[:, self.x_at:self.x_at + W] + self.in_bias[1], self.conv, self.bias)
    S = oracle.gated_unit(u, self.gates[0], self.gate_bias[0], self.gates[1], self.gate_bias[1], self.lam)
    return .7 * S * y

  def state(self, slots=3):
    W, blocks, taps = self.shape
    return state_of(GatedLinearUnit, {"width": W, "blocks": blocks, "conv": taps}, self.kind, slots)

  def run(self, proj, state, step):
    proj, *weights = on_device(self.kind, proj, self.in_bias, self.conv, self.bias, self.gates, self.gate_bias, self.lam)
    y = mo.gated_unit(proj, self.y_at, self.x_at, *weights, GatedLinearUnit.RATE, state, step, out_scale=.7)
    return y.cpu().double()

  def __call__(self, lo, hi, state, step):
    return self.run(self.proj[None, lo:hi], state, step)[0]


@on
@pytest.mark.parametrize("shape", UNIT)
def test_gated_unit(kind, shape):
  T = 70
  op = Unit(kind, shape, T)
  want = op.expected()
  close(op(0, T, op.state(), rows(kind)), want, kind[1])
  for cuts in ((50,), (2, 3, 1, 16, 17), (1, 2), (2,) * 9, ()):
    close(run_cut(op, kind, T, cuts), want, kind[1])


@on
@pytest.mark.parametrize("shape", [(24, 2, 4), (4096, 64, 3)])
def test_gated_unit_rows_are_independent(kind, shape):
  if kind[0] == "cpu" and shape[0] > 100:
    pytest.skip("a launch choice of the GPU path")
  a, b = Unit(kind, shape, 50), Unit(kind, shape, 50, seed=9)
  state = a.state(slots=40)
  for t in state:
    t.fill_(3.0)
  slots, lens = [3, -1, 1] + [-1] * 20, [5, 40, 40] + [1] * 20  # more rows than a tile of decode
  pick = [a, b, b] + [a] * 20
  got = a.run(torch.stack([p.proj[:40] for p in pick]), state, rows(kind, slots=slots, lens=lens))
  wa, wb = a.expected(), b.expected()
  close(got[0, :5], wa[:5], kind[1])
  assert (got[1] == 0).all() and (got[0, 5:] == 0).all()
  close(got[2], wb[:40], kind[1])
  for i in range(8):
    at = [40 + i] + [0] * 20 + [5 + i]
    got = a.run(torch.stack([o.proj[p:p + 1] for o, p in zip([b] + [a] * 21, at)]), state,
                rows(kind, True, positions=at, slots=[1] + [-1] * 20 + [3]))
    close(got[0, 0], wb[40 + i], kind[1])
    assert (got[1:21] == 0).all()
    close(got[21, 0], wa[5 + i], kind[1])
  assert all((t[0] == 3).all() and (t[2] == 3).all() for t in state)


@on
@pytest.mark.parametrize("shape", [(24, 2, 4), (256, 2, 3)])
@pytest.mark.parametrize("cuts", [(), (70,), (250,)])
def test_gated_unit_of_long_prompts_in_segments(kind, shape, cuts):
  """Few channels and many tokens: rows are walked in segments side by side,
  also rows that end in an early one."""
  T = 400
  ops = [Unit(kind, shape, T, seed=s) for s in (0, 9)]
  want = [op.expected() for op in ops]
  state, p = ops[0].state(), 0
  for t in state:
    t.fill_(3.0)
  for n in (*cuts, T - sum(cuts)):
    lens = [n, n if p + n < T else 37]
    got = ops[0].run(torch.stack([o.proj[p:p + n] for o in ops]), state, rows(kind, start=p, slots=[2, 1], lens=lens))
    for g, w, m in zip(got, want, lens):
      close(g[:m], w[p:p + m], kind[1])
      assert (g[m:] == 0).all()
    p += n
  # the short row goes on from the state its own end left
  o, q = ops[1], T - n + 37
  got = o.run(o.proj[None, q:q + 1], state, rows(kind, True, positions=[q], slots=[1]))
  close(got[0], want[1][q:q + 1], kind[1])
  assert all((t[0] == 3.0).all() for t in state)


@on
def test_gated_unit_remembers_far_inputs(kind):
  """Almost no decay, and an input gate that one early token opens."""
  def make():
    op = Unit(kind, (16, 2, 2), 300)
    op.lam = torch.full((16,), -12.0).double()  # a = 1 - 5e-5 at the most
    op.gates[1] = torch.eye(8).double() * 4
    op.gate_bias[1] = -18.0
    op.conv[:, 0], op.conv[:, 1], op.bias, op.in_bias[1] = 0.0, 1.0, torch.zeros(16).double(), 0.0
    return op
  op, without = make(), make()
  op.proj[3, op.x_at:op.x_at + 16] = 6.0
  want = op.expected()
  assert (want - without.expected())[200:].pow(2).mean() > .5 * want[200:].pow(2).mean()
  close(op(0, 300, op.state(), rows(kind)), want, kind[1])
  close(run_cut(op, kind, 300, (2, 64, 33)), want, kind[1])


# ---------------------------------------------------------------- experts

EXPERTS = [  # width, ff, experts, top, shared ff (0: none)
  (72, 40, 12, 3, 0),
  (64, 48, 20, 2, 48),
  (96, 33, 6, 6, 200),    # all of them, and a shared one much wider
  (50, 24, 5, 1, 10),
  (128, 64, 8, 8, 64),
  (64, 16, 1, 1, 70),
  (160, 96, 80, 16, 96),
  (64, 24, 4, 2, 1290),   # cut into more pieces than lanes
]


class Experts:
  def __init__(self, kind, shape, seed=0):
    self.kind, self.shape = kind, shape
    D, ff, E, top, shared = shape
    self.m = {"router": {"experts": E, "top": top}, "expert": {"ff": ff}, "shared": {"ff": shared} if shared else None}
    act = {"alpha": 1.0, "limit": float("inf"), "plus": 0.0}
    self.p = {"expert": {"ff": ff, **act}, "router": {**self.m["router"], "weights": "softmax"}, "shared": self.m["shared"]}
    self.w = {"router": rnd(E, D, seed=seed + 1, scale=1.5 * D ** -.5)}
    if shared:
      self.w["shared.sg"] = rnd(1, D, seed=seed + 2, scale=D ** -.5)
    for i, (name, n) in enumerate([(f"e{e}.", ff) for e in range(E)] + ([("shared.", shared)] if shared else [])):
      for j, part in enumerate(("gate", "up")):
        self.w[name + part] = rnd(n, D, seed=seed + 10 + 3 * i + j, scale=1.5 * D ** -.5)
      self.w[name + "down"] = rnd(D, n, seed=seed + 12 + 3 * i, scale=n ** -.5)

  def expected(self, h):
    return oracle.expert_mixture(h, self.w, "", self.m)

  def module(self):
    from xotorch_amd.models.weights import remap_hf_state
    m = GroupedExperts(self.shape[0], self.p)
    m.load_state_dict(remap_hf_state(self.w, m.key_map("", ""), {n: p.shape for n, p in m.named_parameters()}))
    return m.to(self.kind[0], self.kind[1])

  def clear(self, h):
    """Rows of h whose choice does not hang on rounding."""
    D, ff, E, top, shared = self.shape
    z = (h @ self.w["router"].T).sort(descending=True).values
    return h if top == E else h[z[:, top - 1] - z[:, top] > 1e-4]


@on
@pytest.mark.parametrize("shape", EXPERTS)
@pytest.mark.parametrize("tokens", [1, 5, 33, 700])
def test_expert_mixture(kind, shape, tokens):
  """From one token to enough of them for the tiled products; what follows is
  the norm of the output, the stream and what the next sublayer reads."""
  op, D = Experts(kind, shape), shape[0]
  h = op.clear(rnd(min(tokens, 60), D, seed=3))
  again = torch.arange(tokens) % h.shape[0]
  want, h = op.expected(h)[again], h[again]
  x, post, after = rnd(tokens, D, seed=5), rnd(D, seed=6, scale=.3), rnd(D, seed=7, scale=.3)
  hd, pd, nd = on_device(kind, h[None], post, after)
  want = x + oracle.norm_one_plus(want, post, 1e-5)
  module = op.module()
  for following in (nd, mo.STREAM, None):
    with torch.no_grad():
      stream, read = mo.sandwich_norm(module(hd), x[None].to(kind[0], F32), pd, following, 1e-5)
    assert stream.dtype == F32
    close(stream[0].cpu().double() - x, want - x, kind[1])
    if following is None:
      assert read is None
    else:
      assert read.dtype == kind[1]
      close(read[0], want if following is mo.STREAM else oracle.norm_one_plus(want, after, 1e-5), kind[1])


@on
def test_softmax_over_the_chosen_only(kind):
  """Logits far apart and far from zero: nothing overflows, and what is not
  chosen takes no share."""
  op = Experts(kind, (64, 16, 6, 2, 0))
  h = rnd(20, 64, seed=3)
  h[:, 0] = 1.0
  op.w["router"] *= .05
  op.w["router"][:, 0] = torch.tensor([200.0, 199.0, 196.0, -300.0, 0.0, 100.0])
  want = op.expected(h)
  p = torch.softmax(h @ op.w["router"][:2].T, -1)
  alone = sum(p[:, e:e + 1] * oracle.gated_mlp(h, op.w, f"e{e}.") for e in (0, 1))
  close(want, alone, F32)
  (hd,) = on_device(kind, h[None])
  with torch.no_grad():
    got, _ = mo.add_norm(op.module()(hd), torch.zeros(1, 20, 64, device=kind[0]), 1.0, None, 1e-5)
  close(got[0], want, kind[1], 5)  # logits of 200 have a coarser last place


@pytest.mark.gpu
@pytest.mark.parametrize("shape,tokens", [((72, 40, 2, 1, 40), 3000), ((256, 200, 4, 2, 300), 5000)])
def test_large_tiles(shape, tokens):
  """So many tokens per expert that the widest tiles run, with ragged ends."""
  op = Experts(("cuda", BF16), shape)
  h = op.clear(rnd(50, shape[0], seed=3))
  again = torch.arange(tokens) % h.shape[0]
  with torch.no_grad():
    y = op.module()(h[again][None].to("cuda", BF16))
    got, _ = mo.add_norm(y, torch.zeros(1, tokens, shape[0], device="cuda"), 1.0, None, 1e-5)
  close(got[0], op.expected(h)[again], BF16)


@on
@pytest.mark.parametrize("D", [72, 257, 1024, 5000])
def test_output_norm_and_stream(kind, D):
  x, y, b, n = rnd(3, 2, D), rnd(3, 2, D, seed=1, scale=3), rnd(D, seed=3, scale=.3), rnd(D, seed=4, scale=.3)
  yd, bd, nd = on_device(kind, y, b, n)
  want = x + oracle.norm_one_plus(y, b, 1e-5)
  for following in (nd, mo.STREAM):
    got, h = mo.sandwich_norm(yd, x.to(kind[0], F32), bd, following, 1e-5)
    close(got, want, F32)
    assert h.dtype == kind[1] and h.data_ptr() != got.data_ptr() or kind[1] == F32
    close(h, want if following is mo.STREAM else oracle.norm_one_plus(want, n, 1e-5), kind[1])


# ---------------------------------------------------------------- model

def variants():
  one = cases.small(width=64, vocab=37, embedding={"scale": 1.0}, layers=[
    {"type": "attention", "mlp": {"kind": "moe", "expert": {"ff": 64}, "router": {"experts": 1, "top": 1}, "shared": {"ff": 1}},
     "mixer": {"heads": 1, "kv_heads": 1, "dim": 16, "vdim": 16, "scale": 1.0, "softcap": 1.0,
               "mask": {"size": 1, "keep_first": 1},
               "rot": {"base": 10.0, "dims": 2, "scaling": {"factor": 1.0, "low": 1.0, "high": 2.0, "original": 8}}}},
    {"type": "rglru", "mlp": None, "mixer": {"width": 32, "blocks": 1, "conv": 1}},
    {"type": "attention_2", "mlp": {"kind": "dense", "ff": 1}, "mixer": {
      "heads": 1, "kv_heads": 1, "dim": 8, "vdim": 8, "scale": 1.0, "diff": 0.0, "rot": {"base": 10.0, "dims": 8}}}])
  back = cases.small(norm={"eps": 1e-3}, embedding={"scale": 0.4})
  back["layers"] = back["layers"][::-1]
  for layer in back["layers"]:
    if layer["mixer"].get("kv_from") is not None:
      layer["mixer"].pop("kv_from")
  back["layers"][6]["mixer"]["kv_from"] = 4
  return {"base": cases.small(), "ones": one, "reversed": back}


@pytest.fixture(scope="module")
def checkpoints(tmp_path_factory):
  out = {}
  for name, cfg in variants().items():
    for suffix in ("", "-settled"):
      w = cases.random_weights(cfg, seed=len(name), settled=bool(suffix))
      out[name + suffix] = (write_checkpoint(tmp_path_factory.mktemp("tapupel") / name, cfg, w), cfg, w)
  return out


TOKENS = torch.randint(0, 37, (90,), generator=torch.Generator().manual_seed(3))


@pytest.fixture(scope="module")
def references(checkpoints):
  found = {}

  def get(name, tokens):
    """Logits are causal, so a longer sequence's serve its beginnings."""
    key = tuple(int(t) for t in tokens)
    for (n, other), logits in found.items():
      if n == name and other[:len(key)] == key:
        return logits[:len(key)]
    folder, cfg, w = checkpoints[name]
    found[name, key] = oracle.forward(list(key), w, cfg)
    return found[name, key]
  return get


def near(got, want, dtype):
  close(got, want, dtype, 3)


def case(kind, name):
  """Random routers are full of close calls, which bfloat16 rounding decides
  one way or the other: its runs take routers that settle the choice."""
  return name + "-settled" if kind[1] == BF16 else name


@on
@pytest.mark.parametrize("name", ["base", "ones", "reversed"])
def test_model_whole_cut_and_decoded(kind, name, checkpoints, references):
  want = references(case(kind, name), TOKENS)
  s = Session(kind, checkpoints[case(kind, name)][0])
  near(s.prompt([TOKENS])[0], want, kind[1])
  for cuts in ((2,), (2,) * 10, (33, 1, 31), (1,)):  # the rest token by token: several windows long
    outs, p = [], 0
    for n in cuts:
      outs.append(s.prompt([TOKENS[p:p + n]], p, [2])[0])
      p += n
    for t in range(p, len(TOKENS)):
      outs.append(s.decode([TOKENS[t]], [t], [2]))
    near(torch.cat(outs), want, kind[1])


@on
def test_layers_one_by_one(kind, checkpoints):
  folder, cfg, w = checkpoints[case(kind, "base")]
  want, got = [], []
  oracle.forward(TOKENS[:30].tolist(), w, cfg, layers_out=want)
  s = Session(kind, folder)
  s.prompt([TOKENS[:30]], layers_out=got)
  assert len(got) == len(want) == LAST + 1
  for g, x in zip(got, want):
    near(g[0], x, kind[1])


@on
def test_batch_of_unequal_requests_and_slots_used_again(kind, checkpoints, references):
  name = case(kind, "base")
  s = Session(kind, checkpoints[name][0])
  lens = [1, 40, 7]
  reqs = [TOKENS[:1], TOKENS[10:50], TOKENS[60:67]]
  follow = [TOKENS[20:45], TOKENS[50:75], TOKENS[:25]]
  want = [references(name, torch.cat([a, b])) for a, b in zip(reqs, follow)]
  for slots in ([3, 0, 1], [0, 1, 3], [1, 3, 0]):  # every slot is used by each request in turn
    out = s.prompt(reqs, slots=slots)
    last = s.prompt(reqs, slots=slots, last_only=True)
    got, exp = [], []
    for i, n in enumerate(lens):
      got += [*out[i, :n], last[i]]
      exp += [*want[i][:n], want[i][n - 1]]
    for t in range(25):
      live = [i for i in range(3) if t < 10 or i != 1]  # one ends earlier: its row is parked
      row_slots = [slots[i] if i in live else -1 for i in range(3)]
      out = s.decode([f[t] for f in follow], [n + t for n in lens], row_slots)
      got += [out[i] for i in live]
      exp += [want[i][lens[i] + t] for i in live]
    near(torch.stack(got), torch.stack(exp), kind[1])


@on
def test_prefill_leaves_other_slots_alone(kind, checkpoints):
  s = Session(kind, checkpoints[case(kind, "base")][0])
  s.prompt([TOKENS[:20]], slots=[1])
  before = [t[[0, 1, 3]].clone() for t in s.cache._tensors()]
  s.prompt([TOKENS[:33]], slots=[2])
  s.decode([TOKENS[33], 0], [33, 5], [2, -1])
  assert all((t[[0, 1, 3]] == u).all() for t, u in zip(s.cache._tensors(), before))


@on
def test_a_batch_changes_nothing(kind, checkpoints):
  s = Session(kind, checkpoints[case(kind, "base")][0])
  alone = s.prompt([TOKENS[:50]], slots=[1])[0]
  among = s.prompt([TOKENS[20:27], TOKENS[:50], TOKENS[40:41]], slots=[2, 0, 3])[1]
  near(among, alone, kind[1])


@on
def test_long_decoding(kind, checkpoints, references):
  tokens = TOKENS.repeat(4)[:300]
  want = references(case(kind, "ones"), tokens)
  s = Session(kind, checkpoints[case(kind, "ones")][0], capacity=320)
  got = [s.prompt([tokens[:2]], slots=[1])[0]]
  got += [s.decode([tokens[t]], [t], [1]) for t in range(2, 300)]
  near(torch.cat(got), want, kind[1])


@on
@pytest.mark.parametrize("capacity", [12, 25])  # fewer rows than the windows and their first tokens
def test_capacity_below_the_window(kind, capacity, checkpoints, references):
  s = Session(kind, checkpoints[case(kind, "base")][0], capacity=capacity)
  want = references(case(kind, "base"), TOKENS[:capacity])
  got = [s.prompt([TOKENS[:8]])[0]] + [s.decode([TOKENS[t]], [t]) for t in range(8, capacity)]
  near(torch.cat(got), want, kind[1])


@on
@pytest.mark.parametrize("cut", [1, 2, 4, 7])  # around the layer whose keys and values others read, and its readers
def test_shards_pass_the_stream_and_what_others_read(kind, cut, checkpoints, references):
  folder = checkpoints[case(kind, "base")][0]
  a, b = Session(kind, folder, layers=(0, cut - 1)), Session(kind, folder, layers=(cut, LAST))
  want = references(case(kind, "base"), TOKENS[:40])
  with torch.inference_mode():
    x = TOKENS[None, :30].to(kind[0])
    mid = a.model(x, a.cache.caches, torch.arange(30), 0)
    assert mid.dtype == a.model.hidden_dtype == F32 and mid.shape[-1] == a.model.cfg.hidden_dim == 72 + 80 + 24
    kept_ = mid.clone()
    got = [b.model(mid, b.cache.caches, torch.arange(30), 0, last_only=False)[0]]
    assert (mid == kept_).all()
    mid = a.model(TOKENS[None, 30:39].to(kind[0]), a.cache.caches, torch.arange(30, 39), 30)
    got.append(b.model(mid, b.cache.caches, torch.arange(30, 39), 30, last_only=False)[0])
    pos = torch.tensor([39], dtype=torch.int32, device=kind[0])
    mid = a.model(TOKENS[None, 39:40].to(kind[0]), a.cache.caches, pos, -1, is_decode=True)
    got.append(b.model(mid, b.cache.caches, pos, -1, is_decode=True))
  near(torch.cat(got), want, kind[1])


def test_cacheless_forward_trains(checkpoints, references):
  model = load_model(checkpoints["base"][0])
  out = model(TOKENS[None, :20], None, torch.arange(20), 0, last_only=False)
  close(out[0], references("base", TOKENS[:20]), F32, 3)
  out.float().pow(2).mean().backward()
  dead = [n for n, p in model.named_parameters() if p.grad is None or not p.grad.isfinite().all() or not p.grad.any()]
  assert not dead


# ---------------------------------------------------------------- loading

def test_config(checkpoints):
  folder, raw, _ = checkpoints["base"]
  cfg = config_from_hf(folder / "config.json", "m")
  assert cfg.model_type == "tapupel" and cfg.n_layers == LAST + 1 and cfg.dim == 72 and cfg.norm_eps == 1e-5
  assert cfg.embed_scale == 1.7 and cfg.carried == {"kv1": 104} and cfg.n_experts == 7
  assert [bool(s.params.get("lent")) for s in cfg.layer_specs] == [i == 1 for i in range(LAST + 1)]
  assert cfg.layer_specs[2].moe is None and not cfg.layer_specs[2].ff and cfg.layer_specs[1].ff == 88
  assert cfg.layer_specs[3].moe["shared"] is None and cfg.layer_specs[0].moe["shared"]["ff"] == 100

  def broken(layer, match, mixer=None, **entry):
    bad = cases.small()
    bad["layers"][layer].update(entry)
    bad["layers"][layer]["mixer"].update(mixer or {})
    with pytest.raises(ValueError, match=match):
      config_from_hf(bad, "m")
  broken(0, "unknown mixer", type="wkv")
  broken(1, "unknown feed-forward", mlp={"kind": "sparse"})
  broken(3, "heads differ", {"vdim": 20})
  for j in (0, 3, 5, 7):  # a recurrence, itself, a later one
    broken(3, "no keys and values", {"kv_from": j})
  broken(7, "no keys and values", {"kv_from": 3})  # has none of its own


def test_parameter_count_matches_the_estimate(checkpoints):
  for name in ("base", "reversed"):
    folder = checkpoints[name][0]
    cfg = config_from_hf(folder / "config.json", "m")
    stored = sum(t.numel() for t in checkpoints[name][2].values())
    assert abs(cfg.estimate_param_bytes() / 2 - stored) / stored < 0.02


def test_loader_names_what_is_missing(tmp_path, checkpoints):
  _, cfg, w = checkpoints["base"]
  for gone in ("l1.mix.k", "l0.mix.conv.b", "l0.mix.ri.b", "l1.mix.lk2", "l1.mix.k.norm", "l2.mix.o", "l0.mlp.e3.up",
               "l0.mlp.shared.down", "l0.mlp.shared.sg", "l1.mlp.down", "final.norm"):
    folder = write_checkpoint(tmp_path / gone, cfg, {n: t for n, t in w.items() if n != gone})
    with pytest.raises(RuntimeError, match="missing weights"):
      load_model(folder)


def test_random_weights_leave_padding_zero():
  from xotorch_amd.models import model_class_for
  from xotorch_amd.models.registry import builtin_config
  from xotorch_amd.models.weights import random_init
  cfg = config_from_hf(builtin_config("tapupel-dummy"), "tapupel-dummy")
  model = model_class_for(cfg)(cfg, Shard("m", 0, 4, 5))
  random_init(model)
  m = model.layers["0"].mlp  # six experts of 40, a shared one of 64 + 8
  assert (m.gate_up[:6, :, 40:] == 0).all() and (m.gate_up[7, :, 8:] == 0).all() and (m.gate_up[..., 80:] == 0).all()
  assert (m.down[:6, :, 40:] == 0).all() and (m.down[7, :, 8:] == 0).all()
  assert (m.gate_up[:6, :, :40, :80] != 0).any(-1).all() and (m.gate_up[6] != 0).any(-1).all()


def test_only_causal_keys_grow_with_the_length(checkpoints):
  cfg = config_from_hf(checkpoints["base"][0] / "config.json", "m")
  small, large = (make_cache(cfg, Shard("m", 0, LAST, LAST + 1), 2, n, F32, "cpu") for n in (64, 1000))
  for lid, (a, b) in enumerate(zip(small.caches, large.caches)):
    same = all(t.shape == u.shape for x, y in zip(a, b) for t, u in zip(x, y))
    assert same == (lid not in (1, 5))
    assert bool(sum(t.numel() for x in a for t in x)) == (lid not in (3, 7))  # readers hold nothing


def test_speculative_decoding_refuses_recurrent_state(checkpoints):
  from xotorch_amd.engine.spec import SpeculativeDecoder
  cfg = config_from_hf(checkpoints["base"][0] / "config.json", "m")
  with pytest.raises(ValueError, match="recurrent"):
    SpeculativeDecoder(None, None, cfg, cfg, "cpu", F32)


# ---------------------------------------------------------------- serving

@on
def test_engine_generates(kind, checkpoints, references):
  from xotorch_amd.download.downloader import NoopShardDownloader
  from xotorch_amd.engine.torch_engine import TorchEngine
  name = case(kind, "base")
  eng = TorchEngine(NoopShardDownloader(checkpoints[name][0]), device=kind[0], dtype=kind[1])
  prompt, whole = TOKENS[:14].numpy(), Shard("m", 0, LAST, LAST + 1)

  async def go(rid):
    out, state = await eng.infer_tensor(rid, whole, prompt[None], {"total_len": 60})
    toks = []
    for _ in range(20):
      toks.append(int((await eng.sample(out, temp=0.0))[0]))
      out, state = await eng.infer_tensor(rid, whole, np.array([[toks[-1]]]), state)
    return toks
  loop = asyncio.new_event_loop()
  toks = loop.run_until_complete(go("a"))
  plausible(toks, prompt, kind[1], lambda t: references(name, t))
  assert loop.run_until_complete(go("b")) == toks


@on
def test_scheduler_serves_more_requests_than_slots(kind, checkpoints, references, monkeypatch):
  """Prompts of unequal length in chunks and batches, decode ticks in between,
  slots handed on."""
  monkeypatch.setattr("xotorch_amd.serve_ring.PREFILL_CHUNK", 16)
  w = make_worker(kind, checkpoints[case(kind, "base")][0])
  reqs = [(f"r{i}", TOKENS[i:i + n].tolist(), m) for i, (n, m) in
          enumerate([(5, 25), (40, 6), (16, 12), (1, 30), (33, 9), (2, 3), (17, 20)])]
  got = serve(w, reqs)
  for rid, ids, n in reqs:
    assert len(got[rid]) == n
    plausible(got[rid], ids, kind[1], lambda t: references(case(kind, "base"), t))


def test_two_rank_ring_serves_the_same_tokens(checkpoints, references):
  reqs = [("a", TOKENS[:20].tolist(), 12), ("b", TOKENS[5:9].tolist(), 15), ("c", TOKENS[:11].tolist(), 4)]
  got = two_ranks_serve(checkpoints["base"][0], reqs)
  for rid, ids, n in reqs:
    assert len(got[rid]) == n
    plausible(got[rid], ids, F32, lambda t: references("base", t))


@on
def test_ring_pipeline_prefill_in_slices(kind, monkeypatch):
  """Batch slices of a prefill address their cache rows by slot."""
  from xotorch_amd.parallel.ring import RingPipeline
  got = []
  for chunk in ("2", "8"):
    monkeypatch.setenv("XOT_PREFILL_CHUNK", chunk)
    ring = RingPipeline("tapupel-dummy", 0, 1, kind[0], kind[1], mb_batch=5, prompt_len=30, max_gen=12)
    ring.capture_tokens = True
    ring.prefill()
    for _ in range(8):
      ring.decode_step()
    got.append(torch.cat(ring.generated[0], dim=1).cpu())
  assert got[0].shape == (5, 9)
  if kind[1] == F32:
    assert (got[0] == got[1]).all()


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [F32, BF16])
def test_captured_decode_steps_replay(dtype, checkpoints):
  """The decode graph, replayed between eager work, against eager steps."""
  kind = ("cuda", dtype)
  w, s = make_worker(kind, checkpoints[case(kind, "base")][0]), Session(kind, checkpoints[case(kind, "base")][0])
  with torch.inference_mode():
    for slot, n in ((0, 20), (2, 35)):
      w._begin_prefill(slot, TOKENS[None, :n].cuda())
      w._prefill_hidden([slot], 0)
      w._activate(slot)
      s.prompt([TOKENS[:n]], slots=[slot])
    for t in range(30):
      toks = [TOKENS[20 + t], TOKENS[35 + t]]
      w.tok_buf[0, 0], w.tok_buf[2, 0] = toks[0].cuda(), toks[1].cuda()
      w.run_decode()
      got = w.logits_buf[[0, 2]].float().cpu()
      w._reset_inactive()
      want = s.decode(toks, [20 + t, 35 + t], [0, 2])
      near(got, want, dtype)


@on
def test_trace_replay(kind, checkpoints, references, tmp_path, monkeypatch, capsys):
  """The replay command: whole, cut and ragged steps, slots given back."""
  from xotorch_amd.engine import trace
  folder = checkpoints[case(kind, "base")][0]
  monkeypatch.setattr("xotorch_amd.serve_ring.PREFILL_CHUNK", 32)
  if kind[0] == "cpu":
    monkeypatch.setattr(torch.cuda, "is_available", lambda: False)
  a, b = TOKENS[:75].tolist(), TOKENS[30:50].tolist()
  steps = [{"entries": [{"id": "a", "tokens": a[:67], "want": [0, 10, 11, 32, 66]}, {"id": "b", "tokens": b[:3], "want": [2]}]}]
  steps += [{"entries": [{"id": "b", "tokens": [b[t]], "want": [0]}] +
             ([{"id": "a", "tokens": [a[64 + t]], "want": [0]}] if t < 8 else [])} for t in range(3, 8)]
  steps += [{"entries": [{"id": "b", "tokens": [b[8]], "want": []}], "end": ["a"]},
            {"entries": [{"id": "b", "tokens": b[9:20], "want": [10]}, {"id": "c", "tokens": a[:40], "want": [39]}], "end": ["b"]}]
  for i, s in enumerate(steps):
    s["step"] = i
  monkeypatch.setattr("sys.stdin", io.StringIO("".join(json.dumps(s) + "\n" for s in steps)))
  dtype = "bfloat16" if kind[1] == BF16 else "float32"
  assert trace.main(["--model", str(folder), "--dtype", dtype, "--out", str(tmp_path), "--max-tokens", "160"]) == 0
  assert [x for x in capsys.readouterr().out.splitlines() if x.startswith("done")] == [f"done {i}" for i in range(len(steps))]
  got, exp = [], []
  tokens, at = {"a": a, "b": b, "c": a[:40]}, {"a": 0, "b": 0, "c": 0}
  for s in steps:
    want = []
    for e in s["entries"]:
      ref = references(case(kind, "base"), torch.tensor(tokens[e["id"]]))
      want += [ref[at[e["id"]] + p] for p in e["want"]]
      at[e["id"]] += len(e["tokens"])
    file = tmp_path / f"{s['step']}.f32"
    assert file.exists() == bool(want)
    if want:
      got.append(torch.from_numpy(np.fromfile(file, "<f4")).view(len(want), -1))
      exp += want
  near(torch.cat(got), torch.stack(exp), kind[1])


def test_cli_runs_a_checkpoint_folder(checkpoints, capsys, monkeypatch):
  from xotorch_amd.cli import build_parser, run_model_cli
  from xotorch_amd.models import registry
  monkeypatch.setattr(registry, "model_cards", dict(registry.model_cards))
  folder = checkpoints["base"][0]
  args = build_parser().parse_args(
    ["run", "my-tapupel", "--model-dir", str(folder), "--prompt", "AB", "--inference-engine", "torch",
     "--discovery-module", "none", "--max-generate-tokens", "5", "--disable-tui"])
  monkeypatch.setenv("XOT_OFFLINE", "1")
  # the folder has no tokenizer: the fallback's ids must fit this vocabulary
  from xotorch_amd.engine.tokenizers import DummyTokenizer
  monkeypatch.setattr(DummyTokenizer, "encode", lambda self, text, **kw: [ord(c) % 100 for c in text])
  asyncio.new_event_loop().run_until_complete(run_model_cli(args))
  assert capsys.readouterr().out.strip()
