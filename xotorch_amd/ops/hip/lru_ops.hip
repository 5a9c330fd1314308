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

// 0.5 z (1 + tanh(sqrt(2/pi) (z + 0.044715 z^3))) as z sigmoid(2 sqrt(2/pi) (..))
DEVINL float gelu_tanh(float z) { return z * sigmoidf(1.5957691216057308f * (z + 0.044715f * z * z * z)); }

// gates before the sigmoid -> decay and what enters the state
DEVINL void decay_of(float zr, float zi, float u, float lam, float rate, float& a, float& x) {
  const float r = 1.f / (1.f + expf(-zr)), i = 1.f / (1.f + expf(-zi));
  const float log_a = -rate * r * (fmaxf(lam, 0.f) + log1pf(expf(-fabsf(lam))));
  a = expf(log_a);
  x = sqrtf(-expm1f(2.f * log_a)) * i * u;
}

// A wave makes both gates of 32 channels of a part for 32 tokens; the block's
// four waves take tokens side by side. u [T, W]; gates [2, parts, n, n].
template <typename T, bool WHOLE>
__global__ __launch_bounds__(256) void gates_kernel(
    const T* __restrict__ u, const T* __restrict__ gates, const T* __restrict__ bias, const T* __restrict__ lam,
    float* __restrict__ decay, float* __restrict__ input, int tokens, UnitArgs a) {
  typedef Frag<T> F;
  const int tiles = (a.n + 31) / 32, part = blockIdx.x / tiles, c0 = blockIdx.x % tiles * 32;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, col = lane & 15, quad = lane >> 4;
  const int t0 = (blockIdx.y * 4 + wave) * 32;
  if (t0 >= tokens) return;
  const T *ur[2], *wr[2][2];
#pragma unroll
  for (int j = 0; j < 2; ++j) {
    ur[j] = u + (size_t)min(t0 + j * 16 + col, tokens - 1) * a.W + part * a.n;
#pragma unroll
    for (int g = 0; g < 2; ++g)
      wr[g][j] = gates + ((size_t)g * a.W + part * a.n + min(c0 + j * 16 + col, a.n - 1)) * a.n;
  }
  floatx4 acc[2][2][2];  // gate, channels, tokens
#pragma unroll
  for (int g = 0; g < 2; ++g)
#pragma unroll
    for (int i = 0; i < 2; ++i)
#pragma unroll
      for (int j = 0; j < 2; ++j) acc[g][i][j] = (floatx4)(0.f);
#pragma unroll 2
  for (int k = quad * F::PER; k - quad * F::PER < a.n; k += F::K) {
    typename F::V uf[2], wf[2][2];
#pragma unroll
    for (int j = 0; j < 2; ++j) {
      uf[j] = ld_frag<T, WHOLE>(ur[j], k, a.n);
#pragma unroll
      for (int g = 0; g < 2; ++g) wf[g][j] = ld_frag<T, WHOLE>(wr[g][j], k, a.n);
    }
#pragma unroll
    for (int g = 0; g < 2; ++g)
#pragma unroll
      for (int i = 0; i < 2; ++i)
#pragma unroll
        for (int j = 0; j < 2; ++j) acc[g][i][j] = mma(wf[g][i], uf[j], acc[g][i][j]);
  }
#pragma unroll
  for (int i = 0; i < 2; ++i) {
    const int cl = c0 + i * 16 + quad * 4, c = part * a.n + cl;
    if (cl >= a.n) continue;
    const bool vec = WHOLE || ((a.n & 3) == 0);
    float br[4], bi[4], lm[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int cc = min(c + r, a.W - 1);
      br[r] = ld(bias + cc);
      bi[r] = ld(bias + a.W + cc);
      lm[r] = ld(lam + cc);
    }
#pragma unroll
    for (int j = 0; j < 2; ++j) {
      const int t = t0 + j * 16 + col;
      if (t >= tokens) continue;
      const size_t at = (size_t)t * a.W + c;
      float uv[4], dv[4], xv[4];
      if (vec) ld4(u + at, uv);
      else
#pragma unroll
        for (int r = 0; r < 4; ++r) uv[r] = cl + r < a.n ? ld(u + at + r) : 0.f;
#pragma unroll
      for (int r = 0; r < 4; ++r) decay_of(acc[0][i][j][r] + br[r], acc[1][i][j][r] + bi[r], uv[r], lm[r], a.rate, dv[r], xv[r]);
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
#pragma unroll 4
  for (int s = 0; s < nseg; ++s) {
    const size_t at = ((size_t)b * nseg + s) * W + c;
    const float own = seg_state[at], d = seg_decay[at];
    seg_state[at] = S;
    S = d * S + own;
  }
}

// Decode: 16 rows x 64 channels of a part. The convolution of the part's
// channels goes through LDS 256 at a time; a wave makes both gates of 16
// channels for all rows.
template <typename T>
__global__ __launch_bounds__(256) void unit_step_kernel(
    const T* __restrict__ proj, const T* __restrict__ in_bias, const T* __restrict__ taps, const T* __restrict__ conv_bias,
    const T* __restrict__ gates, const T* __restrict__ bias, const T* __restrict__ lam, float* __restrict__ state,
    T* __restrict__ ring, T* __restrict__ out, int B, UnitArgs a, Step step) {
  typedef Frag<T> F;
  constexpr int CH = 256, LD = CH + 16 / (int)sizeof(T);
  __shared__ __attribute__((aligned(16))) T us[16][LD];
  __shared__ int slots[16], pos[16];
  const int tiles = (a.n + 63) / 64, part = blockIdx.x / tiles, b0 = blockIdx.y * 16;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, col = lane & 15, quad = lane >> 4;
  const int cl0 = blockIdx.x % tiles * 64 + wave * 16;  // this wave's first channel of the part
  if (threadIdx.x < 16) {
    const int b = b0 + threadIdx.x;
    slots[threadIdx.x] = b < B ? step.slot(b) : -1;
    pos[threadIdx.x] = b < B ? step.first(b) : 0;
  }
  __syncthreads();
  auto conv = [&](int r, int c) {  // u of row r, channel c (of all)
    const int slot = slots[r], p = pos[r];
    if (slot < 0) return 0.f;
    const float ib = ld(in_bias + a.W + c);
    float y = ld(conv_bias + c);
    for (int j = 0; j < a.taps; ++j) {
      const int back = a.taps - 1 - j;
      if (p - back < 0) continue;
      const float x = back ? ld(ring + ((size_t)slot * a.taps + (p - back) % a.taps) * a.W + c)
                           : ld(proj + (size_t)(b0 + r) * a.N + a.x_at + c);
      y += (x + ib) * ld(taps + (size_t)c * a.taps + j);
    }
    return y;
  };
  floatx4 acc[2] = {(floatx4)(0.f), (floatx4)(0.f)};
  const T* wr[2];
#pragma unroll
  for (int g = 0; g < 2; ++g) wr[g] = gates + ((size_t)g * a.W + part * a.n + min(cl0 + col, a.n - 1)) * a.n;
  float uo[4] = {0.f, 0.f, 0.f, 0.f};  // u of this lane's row and channels
  const bool whole = a.n % F::K == 0;
  for (int k0 = 0; k0 < a.n; k0 += CH) {
    const int n = min(CH, a.n - k0);
#pragma unroll 4
    for (int i = threadIdx.x; i < 16 * CH; i += 256) {
      const int r = i / CH, k = i % CH;
      st(&us[r][k], k < n ? conv(r, part * a.n + k0 + k) : 0.f);
    }
    __syncthreads();
    if (cl0 < a.n)
      for (int s = 0; s * F::K < n; ++s) {
        const int k = s * F::K + quad * F::PER;
        const typename F::V uf = *(const typename F::V*)&us[col][k];
#pragma unroll
        for (int g = 0; g < 2; ++g)
          acc[g] = mma(whole ? ld_frag<T, true>(wr[g], k0 + k, a.n) : ld_frag<T, false>(wr[g], k0 + k, a.n), uf, acc[g]);
      }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int k = cl0 + quad * 4 + r - k0;
      if (k >= 0 && k < n) uo[r] = ld(&us[col][k]);
    }
    __syncthreads();
  }
  const int b = b0 + col, slot = slots[col], p = pos[col];
  if (b >= B) return;
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int cl = cl0 + quad * 4 + r, c = part * a.n + cl;
    if (cl >= a.n) continue;
    float o = 0.f;
    if (slot >= 0) {
      float d, x;
      decay_of(acc[0][r] + ld(bias + c), acc[1][r] + ld(bias + a.W + c), uo[r], ld(lam + c), a.rate, d, x);
      float* cell = state + (size_t)slot * a.W + c;
      const float S = p > 0 ? d * *cell + x : x;
      *cell = S;
      // the row of the oldest input: no tap of this step reaches it
      ring[((size_t)slot * a.taps + p % a.taps) * a.W + c] = proj[(size_t)b * a.N + a.x_at + c];
      o = S * gelu_tanh(ld(proj + (size_t)b * a.N + a.y_at + c) + ld(in_bias + c)) * a.out_scale;
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
  const int groups = (tokens + 127) / 128;
  CHK(groups <= 65535);
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
    if (a.n % Frag<T>::K == 0)
      hipLaunchKernelGGL((gates_kernel<T, true>), dim3(tiles, groups), dim3(256), 0, stream, P<T>(u), P<T>(gates), P<T>(bias),
                         P<T>(lam), M<float>(decay), M<float>(input), tokens, a);
    else
      hipLaunchKernelGGL((gates_kernel<T, false>), dim3(tiles, groups), dim3(256), 0, stream, P<T>(u), P<T>(gates), P<T>(bias),
                         P<T>(lam), M<float>(decay), M<float>(input), tokens, a);
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
    hipLaunchKernelGGL((unit_step_kernel<T>), grid, dim3(256), 0, cur_stream(), P<T>(proj), P<T>(in_bias), P<T>(taps),
                       P<T>(conv_bias), P<T>(gates), P<T>(bias), P<T>(lam), M<float>(state), M<T>(ring), M<T>(out), B, a,
                       step);
  });
}

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.def("gated_unit", &gated_unit, "gated linear recurrence of prompt rows");
  m.def("gated_unit_step", &gated_unit_step, "gated linear recurrence, one token a row, from the projections on");
}
