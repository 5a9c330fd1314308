// CDNA4 (gfx950) kernels of gated linear recurrences per channel:
//   r, i = sigmoid(block-diagonal products of u),  log a = -rate r softplus(lam)
//   S = a S + sqrt(1 - a^2) i u,  out = S gelu(y)
// The products run on matrix cores with fp32 accumulation and are not rounded
// on the way to the gates; decays, inputs and the state are fp32.
//   - prompts: gates_kernel makes a and sqrt(1 - a^2) i u of all tokens,
//     unit_scan_kernel walks them, long rows in segments side by side
//   - decode: one kernel from the projections to the gated output, the
//     convolution that makes u included
//
// Two element types: bf16 and fp32. Rows of a step address state by slot
// (struct Step): slot -1 is a parked row, which reads and writes no state and
// yields zeros. A row at position 0 ignores what its slot holds.

#include "common.h"

// width, channels of a part, input row and columns, taps, output row and column
struct UnitArgs { int S, W, n, N, y_at, x_at, taps, K, out_at; float rate, out_scale; };

DEVINL float softplus_of(float lam) { return fmaxf(lam, 0.f) + log1pf(expf(-fabsf(lam))); }

// 1 - exp(-x), x >= 0: the series where the difference would cancel
DEVINL float one_minus_exp(float x) {
  const float series = x * (1.f - x * (1.f / 2) * (1.f - x * (1.f / 3) * (1.f - x * (1.f / 4) * (1.f - x * (1.f / 5) *
                       (1.f - x * (1.f / 6))))));
  return x < 0.25f ? series : 1.f - __expf(-x);
}

// gates before the sigmoid -> decay and what enters the state; most: the
// decay's logarithm at an open gate, negated
DEVINL void decay_of(float zr, float zi, float u, float most, float& a, float& x) {
  const float fall = most * sigmoidf(zr);
  a = __expf(-fall);
  x = __builtin_amdgcn_sqrtf(one_minus_exp(2.f * fall)) * sigmoidf(zi) * u;
}

// A wave makes both gates of 32 channels of a part for GROUPS times 32 tokens;
// the block's four waves take neighbouring channels, so that the tokens they
// read are the same and what they write is contiguous. u [T, W]; gates [2,
// parts, n, n]. HELD: k steps whose gate rows stay in registers (0: none).
constexpr int GROUPS = 4;
template <typename T, bool WHOLE, int HELD>
__global__ __launch_bounds__(256) void gates_kernel(
    const T* __restrict__ u, const T* __restrict__ gates, const T* __restrict__ bias, const T* __restrict__ lam,
    float* __restrict__ decay, float* __restrict__ input, int tokens, UnitArgs a) {
  typedef Frag<T> F;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, col = lane & 15, quad = lane >> 4;
  const int tiles = (a.n + 31) / 32, unit = blockIdx.y * 4 + wave, part = unit / tiles, c0 = unit % tiles * 32;
  if (unit >= a.W / a.n * tiles) return;
  const T* wr[2][2];
#pragma unroll
  for (int j = 0; j < 2; ++j)
#pragma unroll
    for (int g = 0; g < 2; ++g)
      wr[g][j] = gates + ((size_t)g * a.W + part * a.n + min(c0 + j * 16 + col, a.n - 1)) * a.n;
  typename F::V held[HELD ? HELD : 1][2][2];
  if (HELD)
#pragma unroll
    for (int s = 0; s < HELD; ++s)
#pragma unroll
      for (int g = 0; g < 2; ++g)
#pragma unroll
        for (int j = 0; j < 2; ++j) held[s][g][j] = ld_frag<T, WHOLE>(wr[g][j], s * F::K + quad * F::PER, a.n);
  float br[2][4], bi[2][4], most[2][4];
#pragma unroll
  for (int i = 0; i < 2; ++i)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int c = part * a.n + min(c0 + i * 16 + quad * 4 + r, a.n - 1);
      br[i][r] = ld(bias + c);
      bi[i][r] = ld(bias + a.W + c);
      most[i][r] = a.rate * softplus_of(ld(lam + c));
    }
  const bool vec = WHOLE || (a.n & 3) == 0;
  for (int group = 0; group < GROUPS; ++group) {
    const int t0 = (blockIdx.x * GROUPS + group) * 32;
    if (t0 >= tokens) return;
    const T* ur[2];
#pragma unroll
    for (int j = 0; j < 2; ++j) ur[j] = u + (size_t)min(t0 + j * 16 + col, tokens - 1) * a.W + part * a.n;
    float uv[2][2][4];  // u of this lane's channels and tokens
#pragma unroll
    for (int i = 0; i < 2; ++i)
#pragma unroll
      for (int j = 0; j < 2; ++j) {
        const int cl = c0 + i * 16 + quad * 4;
        if (vec) ld4(ur[j] + min(cl, a.n - 4), uv[i][j]);
        else
#pragma unroll
          for (int r = 0; r < 4; ++r) uv[i][j][r] = ld(ur[j] + min(cl + r, a.n - 1));
      }
    floatx4 acc[2][2][2];  // gate, channels, tokens
#pragma unroll
    for (int g = 0; g < 2; ++g)
#pragma unroll
      for (int i = 0; i < 2; ++i)
#pragma unroll
        for (int j = 0; j < 2; ++j) acc[g][i][j] = (floatx4)(0.f);
    auto step = [&](const typename F::V (&wf)[2][2], const typename F::V (&uf)[2]) {
#pragma unroll
      for (int g = 0; g < 2; ++g)
#pragma unroll
        for (int i = 0; i < 2; ++i)
#pragma unroll
          for (int j = 0; j < 2; ++j) acc[g][i][j] = mma(wf[g][i], uf[j], acc[g][i][j]);
    };
    if (HELD) {
      typename F::V uf[HELD ? HELD : 1][2];
#pragma unroll
      for (int s = 0; s < HELD; ++s)
#pragma unroll
        for (int j = 0; j < 2; ++j) uf[s][j] = ld_frag<T, WHOLE>(ur[j], s * F::K + quad * F::PER, a.n);
#pragma unroll
      for (int s = 0; s < HELD; ++s) step(held[s], uf[s]);
    } else {
#pragma unroll 2
      for (int k = quad * F::PER; k - quad * F::PER < a.n; k += F::K) {
        typename F::V uf[2], wf[2][2];
#pragma unroll
        for (int j = 0; j < 2; ++j) {
          uf[j] = ld_frag<T, WHOLE>(ur[j], k, a.n);
#pragma unroll
          for (int g = 0; g < 2; ++g) wf[g][j] = ld_frag<T, WHOLE>(wr[g][j], k, a.n);
        }
        step(wf, uf);
      }
    }
#pragma unroll
    for (int j = 0; j < 2; ++j) {
      const int t = t0 + j * 16 + col;
      if (t >= tokens) continue;
#pragma unroll
      for (int i = 0; i < 2; ++i) {
        const int cl = c0 + i * 16 + quad * 4;
        if (cl >= a.n) continue;
        const size_t at = (size_t)t * a.W + part * a.n + cl;
        float dv[4], xv[4];
#pragma unroll
        for (int r = 0; r < 4; ++r)
          decay_of(acc[0][i][j][r] + br[i][r], acc[1][i][j][r] + bi[i][r], uv[i][j][r], most[i][r], dv[r], xv[r]);
        if (vec) {
          st4(decay + at, dv);
          st4(input + at, xv);
        } else
#pragma unroll
          for (int r = 0; r < 4; ++r)
            if (cl + r < a.n) { decay[at + r] = dv[r]; input[at + r] = xv[r]; }
      }
    }
  }
}

// WHOLE walks a row from its state to its end. Where channels and rows are few,
// rows are cut into segments: ENDS walks each from zero and keeps its final
// state and the product of its decays, segment_starts_kernel turns these into
// the states the segments start from, OUTPUTS walks again from there.
enum Pass { WHOLE_ROW, ENDS, OUTPUTS };

// Thread: V channels of one segment, AHEAD tokens in flight.
template <typename T, int V, int PASS>
__global__ __launch_bounds__(256) void unit_scan_kernel(
    const float* __restrict__ decay, const float* __restrict__ input, const T* __restrict__ proj,
    const T* __restrict__ y_bias, float* __restrict__ state, float* __restrict__ seg_state,
    float* __restrict__ seg_decay, T* __restrict__ out, int seg_len, int nseg, UnitArgs a, Step step) {
  constexpr int AHEAD = 8;
  const int c = (blockIdx.x * 256 + threadIdx.x) * V, seg = blockIdx.y, b = blockIdx.z;
  if (c >= a.W) return;
  const int slot = step.slot(b), len = slot < 0 ? 0 : step.len(b, a.S);
  const int lo = seg * seg_len, hi = min(len, lo + seg_len), end = min(a.S, lo + seg_len);
  const size_t tok0 = (size_t)b * a.S, kept = ((size_t)b * nseg + seg) * a.W + c;
  float* cell = state + (size_t)max(slot, 0) * a.W + c;
  float S[V], prod[V], yb[V];
#pragma unroll
  for (int i = 0; i < V; ++i) { S[i] = 0.f; prod[i] = 1.f; }
  if (PASS == WHOLE_ROW && len > 0 && step.start > 0) ldv<V>(cell, S);
  if (PASS == OUTPUTS) ldv<V>(seg_state + kept, S);
  if (PASS != ENDS) ldv<V>(y_bias + c, yb);
  auto walk = [&](int t0, auto count) {  // `count` tokens from t0 on, loads first
    constexpr int N = decltype(count)::value;
    float dv[N][V], xv[N][V], yv[N][V];
#pragma unroll
    for (int j = 0; j < N; ++j) {
      const size_t t = tok0 + t0 + j;
      ldv<V>(decay + t * a.W + c, dv[j]);
      ldv<V>(input + t * a.W + c, xv[j]);
      if (PASS != ENDS) ldv<V>(proj + t * a.N + a.y_at + c, yv[j]);
    }
#pragma unroll
    for (int j = 0; j < N; ++j) {
      float o[V];
#pragma unroll
      for (int i = 0; i < V; ++i) {
        S[i] = dv[j][i] * S[i] + xv[j][i];
        if (PASS == ENDS) prod[i] *= dv[j][i];
        else o[i] = S[i] * gelu_tanh(yv[j][i] + yb[i]) * a.out_scale;
      }
      if (PASS != ENDS) stv<V>(out + (tok0 + t0 + j) * a.K + a.out_at + c, o);
    }
  };
  int t = lo;
  for (; t + AHEAD <= hi; t += AHEAD) walk(t, std::integral_constant<int, AHEAD>());
  for (; t < hi; ++t) walk(t, std::integral_constant<int, 1>());
  if (PASS == ENDS) {
    stv<V>(seg_state + kept, S);
    stv<V>(seg_decay + kept, prod);
    return;
  }
  if (len > lo && len <= lo + seg_len) stv<V>(cell, S);  // the row ends here
#pragma unroll
  for (int i = 0; i < V; ++i) prod[i] = 0.f;
  for (t = max(t, lo); t < end; ++t) stv<V>(out + (tok0 + t) * a.K + a.out_at + c, prod);  // padding
}

// Final states of the segments (each from zero) -> the states they start from.
__global__ __launch_bounds__(256) void segment_starts_kernel(const float* __restrict__ state, float* __restrict__ seg_state,
                                                             const float* __restrict__ seg_decay, int nseg, int W, Step step) {
  const int c = blockIdx.x * 256 + threadIdx.x, b = blockIdx.y, slot = step.slot(b);
  if (c >= W) return;
  float S = slot >= 0 && step.start > 0 ? state[(size_t)slot * W + c] : 0.f;
  constexpr int AHEAD = 16;  // segments in flight
  for (int s0 = 0; s0 < nseg; s0 += AHEAD) {
    float own[AHEAD], d[AHEAD];
#pragma unroll
    for (int j = 0; j < AHEAD; ++j) {
      const size_t at = ((size_t)b * nseg + min(s0 + j, nseg - 1)) * W + c;
      own[j] = seg_state[at];
      d[j] = seg_decay[at];
    }
#pragma unroll
    for (int j = 0; j < AHEAD; ++j)
      if (s0 + j < nseg) {
        seg_state[((size_t)b * nseg + s0 + j) * W + c] = S;
        S = d[j] * S + own[j];
      }
  }
}

// Decode: 16 rows x 64 channels of a part. The convolution of the part's
// channels goes through LDS 256 at a time; a wave makes both gates of 16
// channels for all rows. What does not hang on the convolution is loaded before
// it. TAPS 0: any number of taps. WHOLE: a part is whole k steps.
template <typename T, int TAPS, bool WHOLE>
__global__ __launch_bounds__(256) void unit_step_kernel(
    const T* __restrict__ proj, const T* __restrict__ in_bias, const T* __restrict__ taps, const T* __restrict__ conv_bias,
    const T* __restrict__ gates, const T* __restrict__ bias, const T* __restrict__ lam, float* __restrict__ state,
    T* __restrict__ ring, T* __restrict__ out, int B, UnitArgs a, Step step) {
  typedef Frag<T> F;
  constexpr int CH = 256, LD = CH + 16 / (int)sizeof(T), PRE = 4;
  __shared__ __attribute__((aligned(16))) T us[16][LD];
  __shared__ int slots[16], pos[16];
  const int tiles = (a.n + 63) / 64, part = blockIdx.x / tiles, b0 = blockIdx.y * 16;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, col = lane & 15, quad = lane >> 4;
  const int cl0 = blockIdx.x % tiles * 64 + wave * 16;  // this wave's first channel of the part
  const int nt = TAPS ? TAPS : a.taps;
  if (threadIdx.x < 16) {
    const int b = b0 + threadIdx.x;
    slots[threadIdx.x] = b < B ? step.slot(b) : -1;
    pos[threadIdx.x] = b < B ? step.first(b) : 0;
  }
  __syncthreads();
  const int b = b0 + col, slot = slots[col], p = pos[col];
  floatx4 acc[2] = {(floatx4)(0.f), (floatx4)(0.f)};
  const T* wr[2];
#pragma unroll
  for (int g = 0; g < 2; ++g) wr[g] = gates + ((size_t)g * a.W + part * a.n + min(cl0 + col, a.n - 1)) * a.n;
  auto gate_row = [&](int g, int k) { return ld_frag<T, WHOLE>(wr[g], k, a.n); };
  // of this lane's row and channels
  float uo[4], br[4], bi[4], most[4], S[4], y[4];
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int c = part * a.n + min(cl0 + quad * 4 + r, a.n - 1);
    uo[r] = 0.f;
    br[r] = ld(bias + c);
    bi[r] = ld(bias + a.W + c);
    most[r] = ld(lam + c);
    S[r] = slot >= 0 && p > 0 ? state[(size_t)slot * a.W + c] : 0.f;
    y[r] = (b < B ? ld(proj + (size_t)b * a.N + a.y_at + c) : 0.f) + ld(in_bias + c);
  }
  for (int k0 = 0; k0 < a.n; k0 += CH) {
    const int n = min(CH, a.n - k0);
    typename F::V wf[PRE][2];
#pragma unroll
    for (int s = 0; s < PRE; ++s)
      if (s * F::K < n)
#pragma unroll
        for (int g = 0; g < 2; ++g) wf[s][g] = gate_row(g, k0 + s * F::K + quad * F::PER);
    // a thread has one of 16 * RUNS channels, and RUNS of the rows
    auto convolve = [&](auto runs) {
      constexpr int RUNS = decltype(runs)::value, BATCH = RUNS < 8 ? RUNS : 8;
      const int k = threadIdx.x % (16 * RUNS), r0 = threadIdx.x / (16 * RUNS), c = part * a.n + k0 + min(k, n - 1);
      const float ib = ld(in_bias + a.W + c), cb = ld(conv_bias + c);
#pragma unroll
      for (int j0 = 0; j0 < RUNS; j0 += BATCH) {
        float v[BATCH];
        auto tap = [&](int back) {  // of all rows of the batch, loads first
          float x[BATCH];
#pragma unroll
          for (int j = 0; j < BATCH; ++j) {
            // parked rows load something valid, so that no load waits for a branch
            const int r = r0 + (j0 + j) * (16 / RUNS), at = max(slots[r], 0);
            x[j] = back ? ld(ring + ((size_t)at * nt + max(pos[r] - back, 0) % nt) * a.W + c)
                        : ld(proj + (size_t)min(b0 + r, B - 1) * a.N + a.x_at + c);
          }
          const float w = ld(taps + (size_t)c * nt + nt - 1 - back);
#pragma unroll
          for (int j = 0; j < BATCH; ++j)
            if (pos[r0 + (j0 + j) * (16 / RUNS)] >= back) v[j] += (x[j] + ib) * w;
        };
#pragma unroll
        for (int j = 0; j < BATCH; ++j) v[j] = cb;
        if (TAPS) {
#pragma unroll
          for (int back = 0; back < TAPS; ++back) tap(back);
        } else
          for (int back = 0; back < nt; ++back) tap(back);
#pragma unroll
        for (int j = 0; j < BATCH; ++j) {
          const int r = r0 + (j0 + j) * (16 / RUNS);
          st(&us[r][k], slots[r] >= 0 && k < n ? v[j] : 0.f);
        }
      }
    };
    if (n <= 32) convolve(std::integral_constant<int, 2>());
    else if (n <= 64) convolve(std::integral_constant<int, 4>());
    else if (n <= 128) convolve(std::integral_constant<int, 8>());
    else convolve(std::integral_constant<int, 16>());
    __syncthreads();
    if (cl0 < a.n) {
#pragma unroll
      for (int s = 0; s < PRE; ++s)
        if (s * F::K < n) {
          const typename F::V uf = *(const typename F::V*)&us[col][s * F::K + quad * F::PER];
#pragma unroll
          for (int g = 0; g < 2; ++g) acc[g] = mma(wf[s][g], uf, acc[g]);
        }
#pragma unroll 2
      for (int s = PRE; s * F::K < n; ++s) {
        const int at = s * F::K + quad * F::PER;
        const typename F::V uf = *(const typename F::V*)&us[col][at];
#pragma unroll
        for (int g = 0; g < 2; ++g) acc[g] = mma(gate_row(g, k0 + at), uf, acc[g]);
      }
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int own = cl0 + quad * 4 + r - k0;
      if (own >= 0 && own < n) uo[r] = ld(&us[col][own]);
    }
    __syncthreads();
  }
  if (b >= B) return;
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int cl = cl0 + quad * 4 + r, c = part * a.n + cl;
    if (cl >= a.n) continue;
    float o = 0.f;
    if (slot >= 0) {
      float d, x;
      decay_of(acc[0][r] + br[r], acc[1][r] + bi[r], uo[r], a.rate * softplus_of(most[r]), d, x);
      const float now = d * S[r] + x;
      state[(size_t)slot * a.W + c] = now;
      // the row of the oldest input: no tap of this step reaches it
      ring[((size_t)slot * nt + p % nt) * a.W + c] = proj[(size_t)b * a.N + a.x_at + c];
      o = now * gelu_tanh(y[r]) * a.out_scale;
    }
    st(out + (size_t)b * a.K + a.out_at + c, o);
  }
}

// ===========================================================================
// host side
// ===========================================================================

static UnitArgs unit_args(const Tensor& proj, const Tensor& in_bias, const Tensor& gates, const Tensor& bias,
                          const Tensor& lam, const Tensor& state, const Tensor& out, int64_t y_at, int64_t out_at,
                          double rate, double out_scale, const OptT& slots) {
  const auto dt = io_type(proj);
  for (const Tensor& t : {in_bias, gates, bias, lam, out}) check_io(t, dt);
  check_io(state, torch::kFloat32);
  const int B = proj.size(0), S = proj.size(1), W = lam.numel();
  CHK(proj.dim() == 3 && out.dim() == 3 && out.size(0) == B && out.size(1) == S);
  CHK(gates.dim() == 4 && gates.size(0) == 2 && gates.size(2) == gates.size(3) && gates.size(1) * gates.size(2) == W);
  CHK(in_bias.numel() == 2 * W && bias.numel() == 2 * W && state.dim() == 2 && state.size(1) == W);
  CHK(y_at >= 0 && y_at + W <= proj.size(2) && out_at >= 0 && out_at + W <= out.size(2) && (slots || B <= state.size(0)));
  CHK(B <= 65535);
  return UnitArgs{S, W, (int)gates.size(2), (int)proj.size(2), (int)y_at, 0, 0, (int)out.size(2), (int)out_at,
                  (float)rate, (float)out_scale};
}

// u [B,S,W]: the convolution's output; y: W columns of proj [B,S,N] from y_at on
void gated_unit(Tensor u, Tensor proj, int64_t y_at, Tensor in_bias, Tensor gates, Tensor bias, Tensor lam, double rate,
                Tensor state, OptT slots, OptT lens, int64_t start, Tensor out, int64_t out_at, double out_scale) {
  const UnitArgs a = unit_args(proj, in_bias, gates, bias, lam, state, out, y_at, out_at, rate, out_scale, slots);
  const auto dt = io_type(u);
  const int B = proj.size(0), S = a.S, W = a.W;
  CHK(dt == proj.scalar_type() && u.dim() == 3 && u.size(0) == B && u.size(1) == S && u.size(2) == W);
  if (B == 0 || S == 0) return;
  CHK((int64_t)B * S < INT_MAX / 2);
  const Step step = make_step(slots, c10::nullopt, lens, start, false, B);
  const hipStream_t stream = cur_stream();
  const int tokens = B * S, tiles = W / a.n * ((a.n + 31) / 32);
  auto decay = f32(u, {B, S, W}), input = f32(u, {B, S, W});
  const dim3 gate_grid((tokens + 32 * GROUPS - 1) / (32 * GROUPS), (tiles + 3) / 4);
  CHK(gate_grid.y <= 65535);
  const int V = ((W | a.N | a.y_at | a.K | a.out_at) & 3) == 0 ? 4 : 1;
  // segments where rows and channels are too few to hide the loads
  const int64_t threads = (int64_t)B * (W / V);
  int nseg = threads >= 65536 ? 1 : (int)std::max<int64_t>(1, std::min<int64_t>(S / 32, (65536 + threads - 1) / threads));
  const int seg = (S + nseg - 1) / nseg;
  nseg = (S + seg - 1) / seg;
  Tensor seg_state, seg_decay;
  if (nseg > 1) {
    seg_state = f32(u, {B, nseg, W});
    seg_decay = f32(u, {B, nseg, W});
  }
  float *ss = nseg > 1 ? M<float>(seg_state) : nullptr, *sd = nseg > 1 ? M<float>(seg_decay) : nullptr;
  const dim3 grid((W + 256 * V - 1) / (256 * V), nseg, B);
#define SCAN(V, PASS)                                                                                                 \
  hipLaunchKernelGGL((unit_scan_kernel<T, V, PASS>), grid, dim3(256), 0, stream, P<float>(decay), P<float>(input),     \
                     P<T>(proj), P<T>(in_bias), M<float>(state), ss, sd, M<T>(out), seg, nseg, a, step)
#define SCANS(V)                                                                                                      \
  if (nseg == 1) SCAN(V, WHOLE_ROW);                                                                                  \
  else {                                                                                                              \
    SCAN(V, ENDS);                                                                                                    \
    hipLaunchKernelGGL(segment_starts_kernel, dim3((W + 255) / 256, B), dim3(256), 0, stream, P<float>(state), ss, sd, \
                       nseg, W, step);                                                                                \
    SCAN(V, OUTPUTS);                                                                                                 \
  }
  BY_TYPE(dt, {
    auto make = [&](auto kernel) {
      hipLaunchKernelGGL(kernel, gate_grid, dim3(256), 0, stream, P<T>(u), P<T>(gates), P<T>(bias), P<T>(lam),
                         M<float>(decay), M<float>(input), tokens, a);
    };
    if (a.n == 4 * Frag<T>::K) make(gates_kernel<T, true, 4>);
    else if (a.n % Frag<T>::K == 0) make(gates_kernel<T, true, 0>);
    else make(gates_kernel<T, false, 0>);
    if (V == 4) { SCANS(4) } else { SCANS(1) }
  });
#undef SCANS
#undef SCAN
}

// One token a row: proj [B,1,N] with W columns from x_at (convolved) and y_at on
void gated_unit_step(Tensor proj, int64_t y_at, int64_t x_at, Tensor in_bias, Tensor taps, Tensor conv_bias, Tensor gates,
                     Tensor bias, Tensor lam, double rate, Tensor state, Tensor ring, OptT slots, OptT positions,
                     Tensor out, int64_t out_at, double out_scale) {
  UnitArgs a = unit_args(proj, in_bias, gates, bias, lam, state, out, y_at, out_at, rate, out_scale, slots);
  const auto dt = io_type(proj);
  for (const Tensor& t : {taps, conv_bias, ring}) check_io(t, dt);
  const int B = proj.size(0);
  CHK(a.S == 1 && x_at >= 0 && x_at + a.W <= a.N && taps.dim() == 2 && taps.size(0) == a.W && conv_bias.numel() == a.W);
  CHK(ring.dim() == 3 && ring.size(0) == state.size(0) && ring.size(1) == taps.size(1) && ring.size(2) == a.W);
  if (B == 0) return;
  a.x_at = x_at;
  a.taps = taps.size(1);
  const Step step = make_step(slots, positions, c10::nullopt, 0, true, B);
  const dim3 grid(a.W / a.n * ((a.n + 63) / 64), (B + 15) / 16);
  BY_TYPE(dt, {
    auto run = [&](auto kernel) {
      hipLaunchKernelGGL(kernel, grid, dim3(256), 0, cur_stream(), P<T>(proj), P<T>(in_bias), P<T>(taps), P<T>(conv_bias),
                         P<T>(gates), P<T>(bias), P<T>(lam), M<float>(state), M<T>(ring), M<T>(out), B, a, step);
    };
    const bool whole = a.n % Frag<T>::K == 0;
    if (a.taps == 4) whole ? run(unit_step_kernel<T, 4, true>) : run(unit_step_kernel<T, 4, false>);
    else whole ? run(unit_step_kernel<T, 0, true>) : run(unit_step_kernel<T, 0, false>);
  });
}

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.def("gated_unit", &gated_unit, "gated linear recurrence of prompt rows");
  m.def("gated_unit_step", &gated_unit_step, "gated linear recurrence, one token a row, from the projections on");
}
