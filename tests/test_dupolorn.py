"""Dupolorn: every mechanism alone, the model through its cache, and serving,
against the plain functions of dupolorn_oracle.py. CPU runs take the torch path
in 32-bit, GPU runs the HIP kernels in 32-bit and bfloat16."""
import asyncio
import io
import json

import numpy as np
import pytest
import torch

import dupolorn_cases as cases
import dupolorn_oracle as oracle
from layered_common import (
  BF16, F32, Session, close, load_model, make_worker, on, on_device, plausible, rnd, rows, run_cut, serve, state_of,
  two_ranks_serve, write_checkpoint,
)
from xotorch_amd.engine.kvcache import make_cache
from xotorch_amd.models.config import config_from_hf
from xotorch_amd.models.experts import GroupedExperts
from xotorch_amd.models.llama import XotLinear
from xotorch_amd.models.mixers import LatentAttention, MatrixMemory, turn_rates
from xotorch_amd.ops import mixer_ops as mo
from xotorch_amd.shard import Shard

LAST = len(cases.BASE["layers"]) - 1


# ---------------------------------------------------------------- embedding

PAIRS = {"buckets": 37, "mul_prev": 5, "mul_cur": 3}


class Embedding:
  def __init__(self, kind, T, D=24, rule=PAIRS, vocab=50, seed=0):
    self.kind, self.rule = kind, rule
    self.tokens = torch.randint(0, vocab, (T,), generator=torch.Generator().manual_seed(seed))
    self.w = {"embed": rnd(vocab, D, seed=1), "bigram": rnd(rule["buckets"] + 1, D, seed=2)}

  def expected(self):
    return oracle.embed(self.tokens.tolist(), self.w, {"scale": 1.5, "bigram": self.rule})

  def state(self, slots=3):
    return (torch.zeros(slots, 1, dtype=torch.int32, device=self.kind[0]),)

  def run(self, tokens, state, step):
    table, pairs = on_device(self.kind, self.w["embed"], self.w["bigram"])
    step.depth = mo.Depth(table, tokens.shape, 1)
    x = mo.embed_pairs(tokens.to(self.kind[0]), table, 1.5, pairs, self.rule, state[0], step)
    assert x.dtype == F32 and x is step.depth.streams[0]
    return x.cpu().double()

  def __call__(self, lo, hi, state, step):
    return self.run(self.tokens[None, lo:hi], state, step)[0]


@on
@pytest.mark.parametrize("D,rule", [(24, PAIRS), (70, {"buckets": 1, "mul_prev": 1, "mul_cur": 1}),
                                    (1030, {"buckets": 4093, "mul_prev": 100003, "mul_cur": 77})])
def test_pairs_are_embedded_across_cuts(kind, D, rule):
  op = Embedding(kind, 40, D, rule)
  want = op.expected()
  close(op(0, 40, op.state(), rows(kind)), want, F32)
  for cuts in ((1, 2, 4, 3), (2,) * 7, (39,), ()):
    close(run_cut(op, kind, 40, cuts), want, F32)


@on
def test_the_first_token_has_a_row_of_its_own(kind):
  """What a slot held before does not count; equal pairs are equal wherever they
  stand, and the order within a pair matters."""
  op = Embedding(kind, 4)
  op.tokens = torch.tensor([7, 9, 7, 9])
  got = op(0, 4, op.state(), rows(kind))
  assert (got[1] == got[3]).all() and not torch.equal(got[0], got[2])
  op.w["bigram"][-1] += 100.0
  again = op(0, 4, op.state(), rows(kind))
  assert (again[0] != got[0]).all() and (again[1:] == got[1:]).all()


@on
def test_pairs_of_unequal_rows(kind):
  a, b = Embedding(kind, 30), Embedding(kind, 30, seed=5)
  state, wa, wb = a.state(4), a.expected(), b.expected()
  state[0].fill_(11)
  got = a.run(torch.stack([a.tokens[:20], b.tokens[:20], b.tokens[:20]]), state, rows(kind, slots=[3, -1, 1], lens=[4, 20, 20]))
  close(got[0, :4], wa[:4], F32)
  close(got[2], wb[:20], F32)
  for i in range(10):
    at = [20 + i, 0, 4 + i]
    got = a.run(torch.stack([o.tokens[p:p + 1] for o, p in zip((b, a, a), at)]), state,
                rows(kind, True, positions=at, slots=[1, -1, 3]))
    close(got[0, 0], wb[20 + i], F32)
    close(got[2, 0], wa[4 + i], F32)
  assert state[0][0] == 11 and state[0][2] == 11


# ---------------------------------------------------------------- a layer's end

class Ending:
  """Sublayer outputs joining the stream, the average over depth, two norms and
  the convolution of the first, for T tokens."""

  def __init__(self, kind, T, D, done, taps, seed=0):
    self.kind, self.T, self.D, self.done = kind, T, D, done
    self.streams = [rnd(T, D, seed=seed + 10 + j) for j in range(done)]
    self.x, self.y, self.z = (rnd(T, D, seed=seed + i) for i in range(3))
    self.average, self.g = rnd(done + 1, seed=seed + 4), torch.tensor([1.25, -.5]).double()
    self.taps = rnd(D, taps, seed=seed + 5, scale=.5)

  def expected(self, z=True):
    new = self.x + self.y + (self.z if z else 0)
    x = oracle.depth_average([*self.streams, new], self.average)
    h = [oracle.rms(x, 1e-5) * g for g in self.g]
    return torch.cat([new, x, oracle.with_conv(h[0], self.taps), h[1]], dim=-1)

  def state(self, slots=3):
    n = self.taps.shape[1]
    return (torch.zeros(slots, n, self.D, dtype=self.kind[1], device=self.kind[0]),)

  def run(self, ops, los, hi, state, step, z=True):
    dev = self.kind[0]
    def rows_of(pick):
      parts = [pick(o)[lo:h] for o, lo, h in zip(ops, los, hi)]
      return torch.stack([torch.nn.functional.pad(p, (0, 0, 0, max(len(q) for q in parts) - len(p))) for p in parts])
    x = rows_of(lambda o: o.x).to(dev, F32)
    y, zz, g1, g2, avg, taps = on_device(self.kind, rows_of(lambda o: o.y), rows_of(lambda o: o.z), *self.g, self.average,
                                         self.taps)
    step.depth = mo.Depth(x, x.shape[:-1], self.done + 1, self.D)
    for j in range(self.done):
      step.depth.add(rows_of(lambda o: o.streams[j]).to(dev, F32))
    x, h = mo.depth_norm(y, zz if z else None, x, avg, mo.Reads((g1, g2), taps, state[0]), 1e-5, self.kind[1], step)
    assert x.dtype == F32 and h[0].dtype == h[1].dtype == self.kind[1] and len(step.depth.streams) == self.done + 1
    return [t.cpu().double() for t in (step.depth.streams[-1], x, *h)]

  def __call__(self, lo, hi, state, step):
    return torch.cat(self.run([self], [lo], [hi], state, step), dim=-1)[0]

  def check(self, got, want):
    """The streams are fp32 in either type."""
    D = self.D
    close(got[..., :2 * D], want[..., :2 * D], F32)
    close(got[..., 2 * D:], want[..., 2 * D:], self.kind[1])


@on
@pytest.mark.parametrize("D,done,taps", [(72, 1, 3), (50, 3, 4), (257, 4, 1), (1024, 9, 2), (3000, 6, 6), (36, 17, 4),
                                          (40, 64, 2), (2048, 150, 4), (5000, 3, 2)])
def test_layer_end(kind, D, done, taps):
  op = Ending(kind, 24, D, done, taps)
  want = op.expected()
  op.check(op(0, 24, op.state(), rows(kind)), want)
  for cuts in ((1, 2, 9), (2,) * 6, (23,), ()):
    op.check(run_cut(op, kind, 24, cuts), want)
  alone = torch.cat(op.run([op], [0], [24], op.state(), rows(kind), z=False), dim=-1)[0]
  op.check(alone, op.expected(z=False))


@on
def test_layer_ends_are_independent(kind):
  a, b = Ending(kind, 30, 40, 2, 4), Ending(kind, 30, 40, 2, 4, seed=50)
  b.average, b.taps = a.average, a.taps
  state, wa, wb = a.state(4), a.expected(), b.expected()
  state[0].fill_(3.0)
  got = torch.cat(a.run([a, b, b], [0, 0, 0], [5, 20, 20], state, rows(kind, slots=[3, -1, 1], lens=[5, 20, 20])), dim=-1)
  a.check(got[0, :5], wa[:5])
  a.check(got[2], wb[:20])
  for i in range(8):
    at = [20 + i, 0, 5 + i]
    got = torch.cat(a.run([b, a, a], at, [p + 1 for p in at], state, rows(kind, True, positions=at, slots=[1, -1, 3])), dim=-1)
    a.check(got[0], wb[20 + i:21 + i])
    a.check(got[2], wa[5 + i:6 + i])
  assert (state[0][[0, 2]] == 3).all()


@on
def test_input_convolution_remembers_all_its_taps(kind):
  """One token's input shows in as many outputs as there are taps, whatever part
  of them is decoded."""
  op = Ending(kind, 12, 16, 1, 4)
  for t in (op.x, op.y, op.z, op.streams[0]):
    t[:, 1:] *= 1e-3
    t[:, 0] = 4.0  # fixes the norm
  op.x[5, 3] = 40.0
  op.taps[3] = torch.tensor([8.0, -4.0, 2.0, 1.0])
  want = op.expected()
  spread = want[5:10, 2 * 16 + 3].abs()
  assert (spread[:4] > 20 * spread[4]).all()
  for cuts in ((12,), (6,), (7,), (5, 2), (8,), ()):
    op.check(run_cut(op, kind, 12, cuts), want)


@on
def test_entry_reads_the_stream_alone(kind):
  x, g = rnd(2, 7, 44), rnd(1, seed=3).reshape(())
  (gd,) = on_device(kind, g)
  got, = mo.read_stream(x.to(kind[0], F32), mo.Reads((gd,)), 1e-3, kind[1], rows(kind))
  assert got.dtype == kind[1]
  close(got, oracle.rms(x, 1e-3) * g, kind[1])


# ---------------------------------------------------------------- elementwise

@on
@pytest.mark.parametrize("I", [8, 33, 1030])
def test_gelu_gate(kind, I):
  gu = rnd(3, 2, 2 * I, scale=3.0)
  (d,) = on_device(kind, gu)
  close(mo.gated_packed(d, "gelu_tanh"), oracle.gelu_tanh(gu[..., :I]) * gu[..., I:], kind[1])


@on
@pytest.mark.parametrize("n", [12, 101])
def test_soft_cap(kind, n):
  x = rnd(3, n, scale=20.0)
  (d,) = on_device(kind, x)
  got = mo.soft_cap(d, 7.5)
  assert got.dtype == F32 and got.abs().max() <= 7.5
  close(got, oracle.soft_cap(x, 7.5), F32)


# ---------------------------------------------------------------- latent attention

LATENT = [  # heads, unrotated and rotated dims, values' dim, latent, sink, gate
  (3, 20, 12, 28, 44, True, True),
  (16, 128, 64, 128, 256, True, True),
  (17, 16, 8, 18, 56, True, False),
  (4, 64, 32, 64, 128, False, True),
  (1, 10, 2, 7, 9, True, True),
  (8, 32, 32, 48, 64, False, False),
  (5, 192, 64, 256, 520, True, True),
]


class Latent:
  def __init__(self, kind, shape, T, seed=0):
    self.kind, self.T = kind, T
    self.H, self.d, self.r, self.e, self.R, sink, gate = self.shape = shape
    self.rot, self.scale = {"base": 300.0, "dims": self.r}, 1.5 / (self.d + self.r) ** .5
    nq, nc = self.H * (self.d + self.r), self.R + self.r
    self.q_at, self.c_at = 4, 8 + nq
    self.g_at = self.c_at + nc + 3 if gate else None
    self.proj = rnd(T, self.c_at + nc + 3 + self.H * self.e + 2, seed=seed, scale=1.3)
    self.norm = (rnd(self.R, seed=1) * .2 + 1).to(BF16).double()
    self.uk, self.uv = rnd(self.H * self.d, self.R, seed=2, scale=self.R ** -.5), rnd(self.H * self.e, self.R, seed=3, scale=self.R ** -.5)
    self.sink = rnd(self.H, seed=4, scale=2.0) if sink else None
    self.up = XotLinear(self.R, self.H * (self.d + self.e), bias=False)
    with torch.no_grad():
      self.up.weight.copy_(torch.cat([self.uk, self.uv]))
    self.up = self.up.to(kind[0], kind[1])

  def expected(self):
    m = {"heads": self.H, "dim": self.d, "rot_dim": self.r, "vdim": self.e, "rot": self.rot, "scale": self.scale}
    c = self.proj[:, self.c_at:self.c_at + self.R + self.r]
    o = oracle.latent_attention(self.proj[:, self.q_at:self.q_at + self.H * (self.d + self.r)], c[:, :self.R], c[:, self.R:],
                                self.uk, self.uv, self.norm, m, 1e-5, self.sink)
    if self.g_at is not None:
      o = o * oracle.sigmoid(self.proj[:, self.g_at:self.g_at + self.H * self.e])
    return .7 * o

  def state(self, slots=3, capacity=512):
    return state_of(LatentAttention, {"kv_rank": self.R, "rot_dim": self.r}, self.kind, slots, capacity)

  @torch.no_grad()
  def run(self, x, state, step):
    x, norm = on_device(self.kind, x, self.norm)
    sink = None if self.sink is None else self.sink.to(*self.kind)
    freq = torch.tensor(turn_rates(self.rot), dtype=F32, device=self.kind[0])
    out, width = None, self.H * self.e
    if x.is_cuda:  # columns of a wider tensor
      out = torch.full((*x.shape[:2], (16 + width + 3) // 4 * 4), 9.0, dtype=x.dtype, device=x.device)
    y = mo.latent_attn(x, self.q_at, self.c_at, self.H, self.d, self.r, self.R, self.e, norm, self.up, freq, self.scale, 1e-5,
                       state, step, sink, self.g_at, out=out, out_at=8 if x.is_cuda else 0, out_scale=.7)
    if x.is_cuda:
      assert (y[..., :8] == 9).all() and (y[..., 8 + width:] == 9).all()
      y = y[..., 8:8 + width]
    return y.cpu().double()

  def __call__(self, lo, hi, state, step):
    return self.run(self.proj[None, lo:hi], state, step)[0]


@on
@pytest.mark.parametrize("shape", LATENT, ids=lambda s: "-".join(str(int(v)) for v in s))
def test_latent_attention_portions_and_decode(kind, shape):
  op = Latent(kind, shape, 70)
  want = op.expected()
  close(op(0, 70, op.state(), rows(kind)), want, kind[1], 1.5)
  for cuts in ((1, 2, 31, 3), (2,) * 9, (32, 33), (69,), ()):
    close(run_cut(op, kind, 70, cuts), want, kind[1], 1.5)


def ask(op, query, key, score):
  """The query's score with one key, through the rotated part alone, which is
  zero elsewhere; unrotated parts are zero."""
  q = op.proj[:, op.q_at:op.q_at + op.H * (op.d + op.r)].view(op.T, op.H, op.d + op.r)
  t = op.proj[:, op.c_at + op.R:op.c_at + op.R + op.r]
  q[:], t[:] = 0.0, 0.0
  v = torch.where(torch.arange(op.r) % 3 == 0, 2.0, -1.0).double()[None]
  op.scale = score / v.pow(2).sum().item()
  q[query, :, op.d:] = v
  t[key] = oracle.rotate(v, op.rot, first=query - key).to(BF16).double()


def decoded_and_not(op, kind, query, capacity=512):
  """The query's output in a prompt, right after a cut, two after, and decoded."""
  if query < 500:
    yield op(0, query + 1, op.state(capacity=capacity), rows(kind))[query]
  for cut in (1, 2):
    state, p = op.state(capacity=capacity), query + 1 - cut
    if p > 0:
      op(0, p, state, rows(kind, slots=[1]))
      yield op(p, query + 1, state, rows(kind, start=p, slots=[1]))[-1]
  if query:
    state = op.state(capacity=capacity)
    op(0, query, state, rows(kind, slots=[1]))
    yield op(query, query + 1, state, rows(kind, True, positions=[query], slots=[1]))[0]


@on
@pytest.mark.parametrize("query,key", [(99, 0), (96, 63), (64, 31), (95, 32), (33, 32), (127, 96), (128, 127), (160, 0), (31, 31)])
def test_far_keys_show_and_share_with_the_sink(kind, query, key):
  """A key that outweighs all others, but not the sinks, of which one is as
  strong, one weaker and one stronger; the gate is known."""
  op = Latent(kind, (3, 8, 16, 24, 40, True, True), query + 1)
  ask(op, query, key, 24.0)
  op.sink = torch.tensor([24.0, 20.0, 26.0]).double()
  want = op.expected()[query]
  c = oracle.rms(op.proj[key, op.c_at:op.c_at + op.R], 1e-5) * op.norm
  share = oracle.sigmoid(torch.tensor([0.0, 4.0, -2.0]).double())
  gate = oracle.sigmoid(op.proj[query, op.g_at:op.g_at + 72]).view(3, 24)
  alone = .7 * share[:, None] * (op.uv @ c).view(3, 24) * gate
  assert (want - alone.reshape(-1)).abs().max() < 2e-2  # no other key has a say
  for got in decoded_and_not(op, kind, query):
    close(got, want, kind[1])


@on
def test_a_sink_above_or_below_all_scores(kind):
  """Far above, it leaves nothing; far below, it is not there. It is not scaled."""
  op = Latent(kind, (2, 8, 16, 24, 40, True, False), 40)
  op.sink = torch.tensor([90.0, -90.0]).double()
  want = op.expected()
  plain = Latent(kind, (2, 8, 16, 24, 40, False, False), 40).expected()
  assert want[:, :24].abs().max() < 1e-6 and (want[:, 24:] - plain[:, 24:]).abs().max() < 1e-9
  for cuts in ((40,), (20, 2), ()):
    got = run_cut(op, kind, 40, cuts)
    assert got[:, :24].abs().max() < 1e-6
    close(got[:, 24:], want[:, 24:], kind[1], 1.5)


@on
@pytest.mark.parametrize("shape", [(16, 16, 32, 64, 128, True, True), (3, 8, 16, 18, 40, True, False)])
def test_long_latent_caches_split_over_blocks(kind, shape):
  """Decoding late in a long cache, where several blocks share a row: a sink
  counts once, not once a block."""
  op = Latent(kind, shape, 900)
  op.sink = torch.linspace(3, 7, shape[0]).to(BF16).double()  # as much as hundreds of keys
  want = op.expected()
  state = op.state(capacity=1000)
  op(0, 890, state, rows(kind, slots=[2]))
  got = torch.cat([op(t, t + 1, state, rows(kind, True, positions=[t], slots=[2])) for t in range(890, 900)])
  close(got, want[890:], kind[1], 4)  # angles of hundreds of turns


@on
def test_latent_rows_are_independent(kind):
  shape = (6, 24, 8, 16, 56, True, True)
  a, b = Latent(kind, shape, 90), Latent(kind, shape, 90, seed=7)
  state = a.state(slots=4)
  for t in state:
    t.fill_(3.0)
  before = [t[0].clone() for t in state]
  got = a.run(torch.stack([a.proj[:70], b.proj[:70], b.proj[:70]]), state, rows(kind, slots=[3, -1, 1], lens=[5, 70, 70]))
  wa, wb = a.expected(), b.expected()
  close(got[0, :5], wa[:5], kind[1], 1.5)
  assert (got[1] == 0).all() and (got[0, 5:] == 0).all()
  close(got[2], wb[:70], kind[1], 1.5)
  for i in range(18):
    at = [70 + i, 0, 5 + i]
    got = a.run(torch.stack([op.proj[p:p + 1] for op, p in zip((b, a, a), at)]), state,
                rows(kind, True, positions=at, slots=[1, -1, 3]))
    close(got[0, 0], wb[70 + i], kind[1], 1.5)
    assert (got[1] == 0).all()
    close(got[2, 0], wa[5 + i], kind[1], 1.5)
  assert all((t[0] == u).all() for t, u in zip(state, before))


# ---------------------------------------------------------------- matrix memory

MEMORY = [  # heads, key channels, value channels
  (3, 20, 12), (2, 64, 64), (4, 128, 128), (1, 1, 1), (5, 40, 96), (2, 33, 30), (3, 16, 200), (2, 256, 256), (1, 100, 160),
  (6, 48, 33)]


class Memory:
  """Gates, memory, norm per head and output gate together."""

  def __init__(self, kind, shape, T, seed=0, cap=7.0):
    self.kind, self.T, self.cap = kind, T, cap
    self.H, self.d, self.e = self.shape = shape
    H, widths = self.H, [self.H * self.d] * 2 + [self.H * self.e] * 2 + [self.H] * 2
    self.at, n = [], 4
    for w in widths:
      self.at.append(n)
      n = (n + w + 7) // 8 * 8
    self.proj = rnd(T, n + 4, seed=seed)
    self.bias = torch.stack([rnd(H, seed=1, scale=1.5), rnd(H, seed=2, scale=1.5) + 2]).to(BF16).double()
    self.norm = (rnd(H * self.e, seed=3) * .2 + 1).to(BF16).double()

  def part(self, i, x=None):
    w = (self.H * self.d, self.H * self.d, self.H * self.e, self.H * self.e, self.H, self.H)[i]
    return (self.proj if x is None else x)[:, self.at[i]:self.at[i] + w]

  def logs(self):
    i, f = (oracle.soft_cap(self.part(n) + b, self.cap) for n, b in zip((4, 5), self.bias))
    return i, oracle.log_sigmoid(f)

  def memory(self):
    q, k, v = (self.part(i).reshape(self.T, self.H, -1) for i in range(3))
    return oracle.matrix_memory(q * self.d ** -.5, k, v, *self.logs())

  def expected(self):
    o = oracle.rms(self.memory(), 1e-5).reshape(self.T, -1)
    return .7 * o * self.norm * oracle.sigmoid(self.part(3))

  def state(self, slots=3):
    return state_of(MatrixMemory, {"heads": self.H, "dim": self.d, "vdim": self.e}, self.kind, slots)

  def run(self, proj, state, step):
    proj, bias, norm = on_device(self.kind, proj, self.bias, self.norm)
    out, width = None, self.H * self.e
    if proj.is_cuda:
      out = torch.full((*proj.shape[:2], 8 + width + 3), 9.0, dtype=proj.dtype, device=proj.device)
    y = mo.matrix_memory(proj, self.at, *self.shape, bias, self.cap, norm, 1e-5, state, step, out=out,
                         out_at=8 if proj.is_cuda else 0, out_scale=.7)
    if proj.is_cuda:
      assert (y[..., :8] == 9).all() and (y[..., 8 + width:] == 9).all()
      y = y[..., 8:8 + width]
    return y.cpu().double()

  def __call__(self, lo, hi, state, step):
    return self.run(self.proj[None, lo:hi], state, step)[0]


@on
@pytest.mark.parametrize("shape", MEMORY, ids=lambda s: "-".join(map(str, s)))
def test_matrix_memory(kind, shape):
  if kind[0] == "cpu" and shape[1] > 64:
    pytest.skip("a launch choice of the GPU path")
  T = 150
  op = Memory(kind, shape, T)
  want = op.expected()
  close(op(0, T, op.state(), rows(kind)), want, kind[1], 2)
  for cuts in ((130,), (2, 3, 1, 64, 65), (1, 2), (2,) * 9, (63, 2, 31), ()):
    close(run_cut(op, kind, T, cuts), want, kind[1], 2)


@on
@pytest.mark.parametrize("key", [0, 1, 31, 32, 63, 64, 130])
def test_memory_keeps_a_far_token(kind, key):
  """Hardly any forgetting, and one token whose input gate is wide open among
  closed ones: it is all that later queries find."""
  def make(value):
    op = Memory(kind, (2, 16, 16), 200, cap=12.0)
    op.part(4)[:], op.part(5)[:] = -20.0, 20.0
    op.bias[:] = 0.0
    op.part(4)[key] = 20.0
    op.part(0)[key + 1:] = op.part(1)[key] = 1.0  # nothing but this key is asked for
    op.part(2)[key] = value
    return op
  value = rnd(32, seed=9)
  op = make(value)
  want = op.expected()
  alone = .7 * oracle.rms(value.view(2, 16), 1e-5).reshape(-1) * op.norm * oracle.sigmoid(op.part(3))
  assert (want - alone)[key + 1:].abs().max() < 1e-2
  for cuts in ((200,), (key + 1, 2), (64, 64, 2), (2,) * 5, ()):
    close(run_cut(op, kind, 200, cuts), want, kind[1])


@on
@pytest.mark.parametrize("forget,size", [(-9.0, 2 ** -4), (0.0, 3.0), (9.0, 2 ** -4)])
def test_memory_divides_by_what_is_found_or_by_one(kind, forget, size):
  """From tokens that forget all to ones that keep all, input gates on either end:
  what the queries find is larger here and smaller there than the floor, and
  where next to nothing is, the outputs stay small for the norm's epsilon."""
  op = Memory(kind, (4, 24, 20), 120, cap=9.0)
  op.part(0)[:] *= size
  op.part(5)[:] += forget
  op.part(4)[:, ::2] += 6.0
  op.part(4)[:, 1::2] -= 6.0
  op.part(0)[60:] *= 2 ** -13
  op.proj = op.proj.to(BF16).double()
  # a state's divisor, without the small constant
  q, k = (op.part(i).reshape(120, 4, 24) for i in (0, 1))
  i, f = op.logs()
  n, found = torch.zeros(4, 24).double(), []
  for t in range(120):
    n = torch.exp(f[t])[:, None] * n + torch.exp(i[t])[:, None] * k[t]
    found.append((n * q[t]).sum(-1).abs() * 24 ** -.5)
  found = torch.stack(found)
  assert (found > 1.5).any() and (found < .5).any()
  assert op.memory()[60:, 1::2].pow(2).mean() < 1e-5
  want = op.expected()
  for cuts in ((120,), (64, 50), (70,), ()):
    close(run_cut(op, kind, 120, cuts), want, kind[1], 2)


@on
def test_memory_divisor_has_a_small_constant(kind):
  """With the maximum at a high cap, the floor e^-m is below the constant; outputs
  so small that the norm's epsilon shows their size."""
  op = Memory(kind, (2, 8, 8), 40, cap=16.0)
  op.part(4)[:], op.bias[0] = 400.0, 0.0
  op.part(0)[:] *= 2 ** -25
  op.part(2)[:] *= 2 ** -7
  want = op.expected()
  q, k, v = (op.part(i).reshape(40, 2, 8) for i in range(3))
  i, f = op.logs()
  assert i.min() > 15.9
  # without the constant the outputs would be several times larger
  S, n, m, without = torch.zeros(2, 8, 8).double(), torch.zeros(2, 8).double(), torch.zeros(2).double(), []
  for t in range(40):
    top = torch.maximum(f[t] + m, i[t])
    a, b = torch.exp(f[t] + m - top)[:, None], torch.exp(i[t] - top)[:, None]
    S, n, m = a[:, :, None] * S + b[:, :, None] * k[t][:, :, None] * v[t][:, None], a * n + b * k[t], top
    qt = q[t] * 8 ** -.5
    without.append((S * qt[:, :, None]).sum(1) / torch.maximum((n * qt).sum(-1).abs(), torch.exp(-m))[:, None])
  assert torch.stack(without).pow(2).mean() > 10 * op.memory().pow(2).mean()
  for cuts in ((40,), (20,), ()):
    close(run_cut(op, kind, 40, cuts), want, kind[1], 2)


@on
def test_the_running_maximum_starts_at_zero(kind):
  """Input gates far below zero: the first tokens are divided by one, not by what
  they are relative to each other."""
  op = Memory(kind, (2, 8, 8), 30, cap=11.0)
  op.part(4)[:], op.bias[0] = -20.0, 0.0
  op.part(5)[:], op.bias[1] = 20.0, 0.0
  want = op.expected()
  assert op.memory()[0].abs().max() < 1e-3 and want[0].abs().max() < .2  # e^-11 of a value
  for cuts in ((30,), (2, 2), ()):
    close(run_cut(op, kind, 30, cuts), want, kind[1], 2)


@on
@pytest.mark.parametrize("shape", [(3, 24, 20), (2, 128, 96)])
def test_memory_rows_are_independent(kind, shape):
  a, b = Memory(kind, shape, 100), Memory(kind, shape, 100, seed=9)
  state = a.state(slots=4)
  for t in state:
    t.fill_(3.0)
  got = a.run(torch.stack([a.proj[:80], b.proj[:80], b.proj[:80]]), state, rows(kind, slots=[3, -1, 1], lens=[5, 80, 80]))
  wa, wb = a.expected(), b.expected()
  close(got[0, :5], wa[:5], kind[1], 2)
  assert (got[1] == 0).all() and (got[0, 5:] == 0).all()
  close(got[2], wb[:80], kind[1], 2)
  for i in range(12):
    at = [80 + i, 0, 5 + i]
    got = a.run(torch.stack([o.proj[p:p + 1] for o, p in zip((b, a, a), at)]), state,
                rows(kind, True, positions=at, slots=[1, -1, 3]))
    close(got[0, 0], wb[80 + i], kind[1], 2)
    assert (got[1] == 0).all()
    close(got[2, 0], wa[5 + i], kind[1], 2)
  assert all((t[[0, 2]] == 3).all() for t in state)


@on
@pytest.mark.parametrize("cuts", [(), (100,), (700,)])
def test_memory_of_long_prompts_in_segments(kind, cuts):
  """Rows are few and long enough to be walked in segments side by side, also a
  row that ends in an early one."""
  if kind[0] == "cpu" and len(cuts):
    pytest.skip("a launch choice of the GPU path")
  T = 900
  ops = [Memory(kind, (2, 24, 20), T, seed=s) for s in (0, 9)]
  for op in ops:
    op.bias[1] += 4  # memories of hundreds of tokens
  want = [op.expected() for op in ops]
  state, p = ops[0].state(), 0
  for t in state:
    t.fill_(3.0)
  for n in (*cuts, T - sum(cuts)):
    lens = [n, n if p + n < T else 37]
    got = ops[0].run(torch.stack([o.proj[p:p + n] for o in ops]), state, rows(kind, start=p, slots=[2, 1], lens=lens))
    for g, w, m in zip(got, want, lens):
      close(g[:m], w[p:p + m], kind[1], 2)
      assert (g[m:] == 0).all()
    p += n
  # the short row goes on from the state its own end left
  o, q = ops[1], T - n + 37
  for t in range(q, min(q + 3, T)):
    got = o.run(o.proj[None, t:t + 1], state, rows(kind, True, positions=[t], slots=[1]))
    close(got[0], want[1][t:t + 1], kind[1], 2)
  assert all((t[0] == 3.0).all() for t in state)


@pytest.mark.gpu
@pytest.mark.parametrize("tokens", [9000, 17000])
def test_gates_of_rows_with_many_tokens_a_thread(tokens):
  """Chunks of one thread and threads of many chunks: the state after a very long
  prompt is that after its end alone, when memories are short."""
  kind = ("cuda", F32)
  op, tail = Memory(kind, (1, 8, 8), tokens), 300
  op.bias[1] -= 3.0
  got = op(0, tokens, op.state(), rows(kind))
  end = Memory(kind, (1, 8, 8), tail)
  end.bias, end.norm, end.proj = op.bias, op.norm, op.proj[-tail:]
  close(got[-100:], end.expected()[-100:], F32, 5)


# ---------------------------------------------------------------- experts

EXPERTS = [  # width, ff, experts, top, shared ff (0: none)
  (72, 40, 12, 3, 0),
  (64, 48, 20, 2, 48),
  (96, 33, 6, 6, 200),    # all of them, and a shared one much wider
  (50, 24, 5, 1, 10),
  (128, 64, 8, 8, 64),
  (64, 16, 1, 1, 70),
  (160, 96, 80, 16, 96),
  (256, 300, 3, 2, 520),
]


class Experts:
  def __init__(self, kind, shape, seed=0):
    self.kind, self.shape = kind, shape
    D, ff, E, top, shared = shape
    self.m = {"router": {"experts": E, "top": top}, "expert": {"ff": ff}, "shared": {"ff": shared} if shared else None}
    self.p = {"expert": {"ff": ff, "act": "relu2"}, "shared": {"ff": shared, "gated": False} if shared else None,
              "router": {**self.m["router"], "corrected": False, "applied": "input"}}
    self.w = {"router": rnd(E, D, seed=seed + 1, scale=1.5 * D ** -.5)}
    for i, (name, n) in enumerate([(f"e{e}.", ff) for e in range(E)] + ([("shared.", shared)] if shared else [])):
      self.w[name + "up"] = rnd(n, D, seed=seed + 10 + 2 * i, scale=1.5 * D ** -.5)
      self.w[name + "down"] = rnd(D, n, seed=seed + 11 + 2 * i, scale=n ** -.5)

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

  def mixture(self, h):
    """Summed by the kernel that ends a layer."""
    x = torch.zeros(1, *h.shape, device=self.kind[0])
    y = torch.zeros(1, *h.shape, dtype=self.kind[1], device=self.kind[0])
    one, step = torch.ones(1, dtype=self.kind[1], device=self.kind[0]), rows(self.kind)
    step.depth = mo.Depth(x, x.shape[:-1], 1, x.shape[-1])
    with torch.no_grad():
      got, _ = mo.depth_norm(y, self.module()(h[None].to(*self.kind)), x, one, None, 1e-5, self.kind[1], step)
    return got[0]


@on
@pytest.mark.parametrize("shape", EXPERTS)
@pytest.mark.parametrize("tokens", [1, 5, 33, 700])
def test_expert_mixture(kind, shape, tokens):
  """From one token to enough of them for the tiled products."""
  op, D = Experts(kind, shape), shape[0]
  h = op.clear(rnd(min(tokens, 60), D, seed=3))
  again = torch.arange(tokens) % h.shape[0]
  close(op.mixture(h[again]), op.expected(h)[again], kind[1], 1.5)


@on
def test_weights_multiply_the_input(kind):
  """Scores far from one: an activation that is not linear tells whether they
  come before it or after, and they are not made to sum to one."""
  op = Experts(kind, (64, 32, 6, 2, 0))
  h = rnd(20, 64, seed=3)
  h[:, 0] = 1.0
  op.w["router"] *= .05
  op.w["router"][:, 0] = torch.tensor([-1.0, -2.0, -9.0, -9.0, -9.0, -9.0])
  want = op.expected(h)
  z = oracle.sigmoid(h @ op.w["router"].T)
  after = sum(z[:, e:e + 1] * oracle.expert(h, op.w, f"e{e}.") for e in (0, 1))
  assert (want - after).pow(2).mean() > .2 * after.pow(2).mean()
  close(op.mixture(h), want, kind[1], 1.5)


@on
def test_a_shared_expert_has_a_weight_of_one(kind):
  """The routed experts' weights vanish; the shared expert is what is left."""
  op = Experts(kind, (64, 32, 4, 1, 150))
  h = rnd(40, 64, seed=3)
  h[:, 0] = 1.0
  op.w["router"] *= .05
  op.w["router"][:, 0] = -60.0
  want = op.expected(h)
  close(want, oracle.expert(h, op.w, "shared."), F32)
  close(op.mixture(h), want, kind[1], 1.5)


@on
def test_input_weights_through_the_other_sums(kind):
  """The kernels that end other designs' layers take such rows too."""
  op = Experts(kind, (72, 40, 6, 2, 72))
  h, x = op.clear(rnd(30, 72, seed=3)), None
  want = op.expected(h)
  x, post = rnd(1, *h.shape, seed=5), rnd(72, seed=6, scale=.3)
  (hd, pd) = on_device(kind, h[None], post)
  with torch.no_grad():
    got, _ = mo.add_norm(op.module()(hd), x.to(kind[0], F32), 0.5, None, 1e-5)
    close(got[0].cpu().double() - x[0], .5 * want, kind[1], 1.5)
    got, _ = mo.sandwich_norm(op.module()(hd), x.to(kind[0], F32), pd, None, 1e-5)
  close(got[0].cpu().double() - x[0], oracle.rms(want, 1e-5) * (1 + post), kind[1], 1.5)


@pytest.mark.gpu
@pytest.mark.parametrize("shape,tokens", [((72, 40, 2, 1, 40), 3000), ((256, 200, 4, 2, 300), 5000), ((64, 520, 3, 1, 0), 2600)])
def test_large_tiles(shape, tokens):
  """So many tokens per expert that the widest tiles run, with ragged ends."""
  op = Experts(("cuda", BF16), shape)
  h = op.clear(rnd(50, shape[0], seed=3))
  again = torch.arange(tokens) % h.shape[0]
  close(op.mixture(h[again]), op.expected(h)[again], BF16, 1.5)


# ---------------------------------------------------------------- model

def variants():
  one = cases.small(width=64, vocab=37, canon={"taps": 1}, logit_softcap=1.0,
                    embedding={"scale": 1.0, "bigram": {"buckets": 1, "mul_prev": 1, "mul_cur": 1}}, layers=[
    {"type": "latent_attention_2", "mlp": {"kind": "moe", "expert": {"ff": 64}, "router": {"experts": 1, "top": 1}, "shared": {"ff": 1}},
     "mixer": {"heads": 1, "dim": 1, "rot_dim": 2, "vdim": 1, "kv_rank": 1, "scale": 1.0, "rot": {"base": 10.0, "dims": 2}}},
    {"type": "mlstm", "mlp": None, "mixer": {"heads": 1, "dim": 1, "vdim": 6, "gate_cap": 1.0}},
    {"type": "latent_attention", "mlp": {"kind": "dense", "ff": 1}, "mixer": {
      "heads": 1, "dim": 8, "rot_dim": 8, "vdim": 8, "kv_rank": 8, "scale": 1.0, "rot": {"base": 10.0, "dims": 8}}}])
  back = cases.small(norm={"eps": 1e-3}, canon={"taps": 6}, logit_softcap=50.0,
                     embedding={"scale": 0.4, "bigram": {"buckets": 200, "mul_prev": 1009, "mul_cur": 1}})
  back["layers"] = back["layers"][::-1]
  return {"base": cases.small(), "ones": one, "reversed": back}


@pytest.fixture(scope="module")
def checkpoints(tmp_path_factory):
  out = {}
  for name, cfg in variants().items():
    for suffix in ("", "-settled"):
      w = cases.random_weights(cfg, seed=len(name), settled=bool(suffix))
      out[name + suffix] = (write_checkpoint(tmp_path_factory.mktemp("dupolorn") / name, cfg, w), cfg, w)
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
  close(got, want, dtype, 4)


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
  for cuts in ((2,), (2,) * 10, (33, 1, 31), (1,)):
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
def test_every_mechanism_moves_the_logits(kind, checkpoints, references):
  """What the model computes changes with each of the weights that a wrong
  reading could leave out."""
  name = case(kind, "base")
  s = Session(kind, checkpoints[name][0])
  want = s.prompt([TOKENS[:40]])[0]
  params = dict(s.model.named_parameters())
  for tensor in ("embed_pairs.weight", "layers.1.taps", "layers.2.average", "layers.1.mix.branches.only.sink",
                 "layers.0.mix.branches.only.gate_bias", "layers.0.norm2", "norm"):
    keep = params[tensor].detach().clone()
    with torch.no_grad():
      params[tensor].mul_(.3)
    moved = (s.prompt([TOKENS[:40]])[0] - want).pow(2).mean() / want.pow(2).mean()
    with torch.no_grad():
      params[tensor].copy_(keep)
    assert moved > 1e-5, tensor


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
  tokens = TOKENS.repeat(3)[:200]
  want = references(case(kind, "reversed"), tokens)
  s = Session(kind, checkpoints[case(kind, "reversed")][0])
  got = [s.prompt([tokens[:2]], slots=[1])[0]]
  got += [s.decode([tokens[t]], [t], [1]) for t in range(2, 200)]
  near(torch.cat(got), want, kind[1])


@on
@pytest.mark.parametrize("cut", [1, 3, 5])
def test_shards_pass_all_streams(kind, cut, checkpoints, references):
  folder = checkpoints[case(kind, "base")][0]
  a, b = Session(kind, folder, layers=(0, cut - 1)), Session(kind, folder, layers=(cut, LAST))
  want = references(case(kind, "base"), TOKENS[:40])
  with torch.inference_mode():
    x = TOKENS[None, :30].to(kind[0])
    mid = a.model(x, a.cache.caches, torch.arange(30), 0)
    assert mid.dtype == a.model.hidden_dtype == F32 and mid.shape[-1] == a.model.cfg.hidden_dim == 72 * (LAST + 2)
    kept_ = mid.clone()
    got = [b.model(mid, b.cache.caches, torch.arange(30), 0, last_only=False)[0]]
    assert (mid == kept_).all()
    mid = a.model(TOKENS[None, 30:39].to(kind[0]), a.cache.caches, torch.arange(30, 39), 30)
    got.append(b.model(mid, b.cache.caches, torch.arange(30, 39), 30, last_only=False)[0])
    pos = torch.tensor([39], dtype=torch.int32, device=kind[0])
    mid = a.model(TOKENS[None, 39:40].to(kind[0]), a.cache.caches, pos, -1, is_decode=True)
    got.append(b.model(mid, b.cache.caches, pos, -1, is_decode=True))
  near(torch.cat(got), want, kind[1])


@on
def test_three_shards(kind, checkpoints, references):
  """A stage in the middle hands on what it received."""
  folder = checkpoints[case(kind, "base")][0]
  stages = [Session(kind, folder, layers=span) for span in ((0, 0), (1, 3), (4, LAST))]
  with torch.inference_mode():
    x = TOKENS[None, :30].to(kind[0])
    for s in stages:
      x = s.model(x, s.cache.caches, torch.arange(30), 0, last_only=False)
  near(x[0], references(case(kind, "base"), TOKENS[:30]), kind[1])


def test_cacheless_forward_trains(checkpoints, references):
  model = load_model(checkpoints["base"][0])
  out = model(TOKENS[None, :20], None, torch.arange(20), 0, last_only=False)
  close(out[0], references("base", TOKENS[:20]), F32, 4)
  out.float().pow(2).mean().backward()
  dead = [n for n, p in model.named_parameters() if p.grad is None or not p.grad.isfinite().all() or not p.grad.any()]
  assert not dead


@on
def test_cacheless_forward_without_gradients(kind, checkpoints, references):
  name = case(kind, "base")
  model = load_model(checkpoints[name][0], *kind)
  with torch.no_grad():
    out = model(torch.stack([TOKENS[:20], TOKENS[30:50]]).to(kind[0]), None, torch.arange(20), 0, last_only=False)
  near(out[0], references(name, TOKENS[:20]), kind[1])
  near(out[1], references(name, TOKENS[30:50]), kind[1])


# ---------------------------------------------------------------- loading

def test_config(checkpoints):
  folder, raw, _ = checkpoints["base"]
  cfg = config_from_hf(folder / "config.json", "m")
  assert cfg.model_type == "dupolorn" and cfg.n_layers == LAST + 1 and cfg.dim == 72 and cfg.norm_eps == 1e-5
  assert cfg.embed_scale == 1.7 and cfg.final_logit_softcapping == 6.0 and cfg.n_experts == 7
  assert cfg.bigram == {"buckets": 53, "mul_prev": 7, "mul_cur": 11} and cfg.hidden_dim == 72 * (LAST + 2)
  assert [s.conv for s in cfg.layer_specs] == [3] * (LAST + 1)
  assert [bool(s.params.get("sink")) for s in cfg.layer_specs] == [i in (1, 4) for i in range(LAST + 1)]
  assert cfg.layer_specs[3].moe is None and not cfg.layer_specs[3].ff and cfg.layer_specs[2].ff == 88
  assert cfg.layer_specs[0].moe["shared"]["ff"] == 100 and cfg.layer_specs[1].moe["router"]["top"] == 1

  def broken(match, layer=0, **entry):
    bad = cases.small()
    bad["layers"][layer].update(entry)
    with pytest.raises(ValueError, match=match):
      config_from_hf(bad, "m")
  broken("unknown mixer", type="wkv")
  broken("unknown feed-forward", mlp={"kind": "sparse"})
  with pytest.raises(ValueError, match="taps"):
    config_from_hf(cases.small(canon={"taps": 0}), "m")


def test_parameter_count_matches_the_estimate(checkpoints):
  for name in ("base", "reversed"):
    folder = checkpoints[name][0]
    cfg = config_from_hf(folder / "config.json", "m")
    stored = sum(t.numel() for t in checkpoints[name][2].values())
    assert abs(cfg.estimate_param_bytes() / 2 - stored) / stored < 0.02


def test_loader_names_what_is_missing(tmp_path, checkpoints):
  _, cfg, w = checkpoints["base"]
  for gone in ("bigram", "l0.mix.i.b", "l0.mix.f", "l0.mix.norm", "l1.mix.sink", "l1.mix.g", "l1.mix.uk", "l2.mix.dkv.norm",
               "l0.mlp.e3.up", "l0.mlp.shared.down", "l0.mlp.router", "l2.mlp.down", "l3.canon1", "l4.dwa", "l5.norm2",
               "final.norm", "head"):
    folder = write_checkpoint(tmp_path / gone, cfg, {n: t for n, t in w.items() if n != gone})
    with pytest.raises(RuntimeError, match="missing weights"):
      load_model(folder)


def test_every_tensor_is_loaded(checkpoints):
  from xotorch_amd.models.weights import hf_key_map
  folder, _, w = checkpoints["base"]
  cfg = config_from_hf(folder / "config.json", "m")
  assert set(hf_key_map(Shard("m", 0, LAST, LAST + 1), cfg)) == set(w)


def test_random_weights_leave_padding_zero():
  from xotorch_amd.models import model_class_for
  from xotorch_amd.models.registry import builtin_config
  from xotorch_amd.models.weights import random_init
  cfg = config_from_hf(builtin_config("dupolorn-dummy"), "dupolorn-dummy")
  model = model_class_for(cfg)(cfg, Shard("m", 0, cfg.n_layers - 1, cfg.n_layers))
  random_init(model)
  m = model.layers["0"].mlp  # six experts of 40, a shared one of 64 + 8
  assert (m.up[:6, 40:] == 0).all() and (m.up[7, 8:] == 0).all() and (m.up[..., 80:] == 0).all()
  assert (m.down[:6, :, 40:] == 0).all() and (m.down[7, :, 8:] == 0).all()
  assert (m.up[:6, :40, :80] != 0).any(-1).all() and (m.up[6] != 0).any(-1).all()


def test_extensions_are_those_of_the_mixers(checkpoints):
  """What a first run in a fresh checkout compiles."""
  from xotorch_amd.models.registry import builtin_config
  from xotorch_amd.models import model_class_for
  from xotorch_amd.ops.build import EXTENSIONS
  names = {}
  for model in ("dupolorn-dummy", "tapupel-dummy", "lebotar-dummy", "didipel-dummy"):
    cfg = config_from_hf(builtin_config(model), model)
    with torch.device("meta"):
      names[model] = model_class_for(cfg)(cfg, Shard("m", 0, cfg.n_layers - 1, cfg.n_layers)).extensions()
    assert set(names[model]) <= set(EXTENSIONS)
  assert "_hip_mlstm" in names["dupolorn-dummy"] and "_hip_lru" not in names["dupolorn-dummy"]
  assert "_hip_lru" in names["tapupel-dummy"] and "_hip_mlstm" not in names["tapupel-dummy"]


def test_only_latents_grow_with_the_length(checkpoints):
  cfg = config_from_hf(checkpoints["base"][0] / "config.json", "m")
  small, large = (make_cache(cfg, Shard("m", 0, LAST, LAST + 1), 2, n, F32, "cpu") for n in (64, 1000))
  for lid, (a, b) in enumerate(zip(small.caches, large.caches)):
    assert len(a) == (3 if lid == 0 else 2)  # the mixer's, the convolution's, the last token
    same = all(t.shape == u.shape for x, y in zip(a, b) for t, u in zip(x, y))
    assert same == (cfg.layer_specs[lid].mixer == "mlstm")


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
    ring = RingPipeline("dupolorn-dummy", 0, 1, kind[0], kind[1], mb_batch=5, prompt_len=30, max_gen=12)
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
    ["run", "my-dupolorn", "--model-dir", str(folder), "--prompt", "AB", "--inference-engine", "torch",
     "--discovery-module", "none", "--max-generate-tokens", "5", "--disable-tui"])
  monkeypatch.setenv("XOT_OFFLINE", "1")
  # the folder has no tokenizer: the fallback's ids must fit this vocabulary
  from xotorch_amd.engine.tokenizers import DummyTokenizer
  monkeypatch.setattr(DummyTokenizer, "encode", lambda self, text, **kw: [ord(c) % 100 for c in text])
  asyncio.new_event_loop().run_until_complete(run_model_cli(args))
  assert capsys.readouterr().out.strip()
