// CDNA4 (gfx950) kernels of short causal convolutions (also used by other
// recurrences) and of selective state spaces: the scan
//   S[c,n] = exp(dt_c A[c,n]) S[c,n] + dt_c x_c B_n,  y_c = sum_n S[c,n] C_n + D_c x_c
// with the gate y silu(z). Step sizes (softplus), decays and the state are
// fp32; inputs and outputs are bf16 or fp32.
//
// Rows of a step address state by slot (struct Step): slot -1 is a parked row,
// which reads and writes no state and yields zeros. A row at position 0
// ignores what its slot holds.

#include "common.h"

// tokens, channels, input row, first column; add: the input joins its convolution
struct ConvArgs { int S, C, N, at, taps, silu, add; };

constexpr int RUN = 16;  // tokens a thread walks

// Thread: V channels, RUN tokens. TAPS 0: any number of taps, inputs read
// again. in_bias joins the input of every token there is. A decode step also
// stores its input (row p % taps of the ring).
template <typename T, int V, int TAPS>
__global__ __launch_bounds__(256) void short_conv_kernel(
    const T* __restrict__ x, const T* __restrict__ w, const T* __restrict__ bias, const T* __restrict__ in_bias,
    T* __restrict__ ring,
    T* __restrict__ out, ConvArgs a, Step step) {
  const int c = (blockIdx.x * 256 + threadIdx.x) * V, b = blockIdx.z, s0 = blockIdx.y * RUN;
  if (c >= a.C) return;
  const int slot = step.slot(b), len = slot < 0 ? 0 : step.decode ? 1 : step.len(b, a.S);
  const int first = len ? step.first(b) : 0;
  const T* rows = x + (size_t)b * a.S * a.N + a.at + c;
  T* hist = ring + (size_t)max(slot, 0) * a.taps * a.C + c;
  float ib[V];
#pragma unroll
  for (int i = 0; i < V; ++i) ib[i] = 0.f;
  if (in_bias) ldv<V>(in_bias + c, ib);
  auto input = [&](int s, float* o) {  // of token s of this step; s < 0: before it
    if (first + s < 0) {
#pragma unroll
      for (int i = 0; i < V; ++i) o[i] = 0.f;
      return;
    }
    if (s >= 0) ldv<V>(rows + (size_t)s * a.N, o);
    else ldv<V>(hist + (size_t)((first + s) % a.taps) * a.C, o);
#pragma unroll
    for (int i = 0; i < V; ++i) o[i] += ib[i];
  };
  constexpr int NT = TAPS ? TAPS : 1;
  float tw[NT][V], in[NT][V], bs[V];
#pragma unroll
  for (int i = 0; i < V; ++i) bs[i] = 0.f;
  if (bias) ldv<V>(bias + c, bs);
  if (TAPS && s0 < len) {
#pragma unroll
    for (int j = 0; j < NT; ++j)
#pragma unroll
      for (int i = 0; i < V; ++i) tw[j][i] = ld(w + (size_t)(c + i) * TAPS + j);
#pragma unroll
    for (int j = 1; j < NT; ++j) input(s0 - NT + j, in[j]);
  }
  for (int s = s0; s < min(s0 + RUN, a.S); ++s) {
    float y[V];
#pragma unroll
    for (int i = 0; i < V; ++i) y[i] = 0.f;
    if (s < len) {
#pragma unroll
      for (int i = 0; i < V; ++i) y[i] = bs[i];
      if (TAPS) {
#pragma unroll
        for (int j = 0; j + 1 < NT; ++j)
#pragma unroll
          for (int i = 0; i < V; ++i) in[j][i] = in[j + 1][i];
        input(s, in[NT - 1]);
#pragma unroll
        for (int j = 0; j < NT; ++j)
#pragma unroll
          for (int i = 0; i < V; ++i) y[i] += in[j][i] * tw[j][i];
      } else {
        for (int j = 0; j < a.taps; ++j) {
          float v[V];
          input(s - (a.taps - 1 - j), v);
#pragma unroll
          for (int i = 0; i < V; ++i) y[i] += v[i] * ld(w + (size_t)(c + i) * a.taps + j);
        }
      }
      if (a.silu)
#pragma unroll
        for (int i = 0; i < V; ++i) y[i] = siluf(y[i]);
      if (a.add) {
        float v[V];
        input(s, v);
#pragma unroll
        for (int i = 0; i < V; ++i) y[i] += v[i];
      }
      if (step.decode) {
        float v[V];
        ldv<V>(rows, v);
        stv<V>(hist + (size_t)(first % a.taps) * a.C, v);  // the oldest input: no tap reaches it any more
      }
    }
    stv<V>(out + ((size_t)b * a.S + s) * a.C + c, y);
  }
}

// Last inputs of a prompt chunk into the ring.
template <typename T>
__global__ __launch_bounds__(256) void keep_inputs_kernel(const T* __restrict__ x, T* __restrict__ ring, ConvArgs a,
                                                          Step step) {
  const int b = blockIdx.y, slot = step.slot(b), s = step.len(b, a.S) - 1 - blockIdx.x;
  if (slot < 0 || s < 0) return;
  const T* row = x + ((size_t)b * a.S + s) * a.N + a.at;
  T* dst = ring + ((size_t)slot * a.taps + (step.first(b) + s) % a.taps) * a.C;
  for (int i = threadIdx.x; i < a.C; i += 256) dst[i] = row[i];
}

struct ScanArgs {
  int S, C, n;                    // tokens, channels, states
  int zN, z_at, bN, b_at, c_at;   // row lengths and columns of the gate and of B and C
  int K, out_at;
  float out_scale;
  int seg, nseg;                  // tokens of a segment, segments
};

// WHOLE scans a row from its state to its end. With few channels and many
// tokens a row is cut into segments that run side by side: STATES scans each
// from zero and keeps its final state and the sum of its step sizes, from which
// segment_states_kernel makes the state every segment starts from (the decay
// over a segment is exp(A sum dt)), and OUTPUTS scans again from there.
enum Pass { WHOLE, STATES, OUTPUTS };

constexpr float LOG2E = 1.4426950408889634f;

// sum over groups of L lanes (4 or 16), in every lane
template <int L>
DEVINL float lanes_sum(float v) {
  if (L == 16) return row_sum(v);
  v += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0xb1, 0xf, 0xf, true));  // quad_perm 1,0,3,2
  v += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x4e, 0xf, 0xf, true));  // quad_perm 2,3,0,1
  return v;
}

// Prompts. A block scans CH = 256 / L channels; L lanes share a channel, PER
// states each. Tokens come TT at a time: all threads fetch the tile's inputs
// (the next tile's while this one is scanned), step sizes and products go to
// LDS, outputs come back through LDS to be gated and stored in rows.
template <typename T, int L, int PER, int PASS>
__global__ __launch_bounds__(256) void scan_kernel(
    const T* __restrict__ x, const T* __restrict__ pre, const T* __restrict__ bc, const T* __restrict__ z,
    const T* __restrict__ a_log, const T* __restrict__ dt_bias, const T* __restrict__ skip, float* __restrict__ state,
    float* __restrict__ seg_state, float* __restrict__ seg_dt, T* __restrict__ out, ScanArgs a, Step step) {
  constexpr int CH = 256 / L, TT = 16, NP = L * PER, PT = TT * CH / 256, PB = (2 * TT * NP + 255) / 256;
  __shared__ float2 sd[TT][CH];     // dt, dt x
  __shared__ float sb[2][TT][NP];   // B, C
  __shared__ float sy[TT][CH];
  const int c0 = blockIdx.x * CH, b = blockIdx.y, tid = threadIdx.x;
  const int slot = step.slot(b), row_len = slot < 0 ? 0 : step.len(b, a.S), first = step.start;
  // tokens [lo, len) of the row
  const int seg = PASS == WHOLE ? 0 : blockIdx.z, lo = seg * a.seg, len = min(row_len, lo + a.seg);
  const int ch = tid / L, part = tid % L, c = c0 + ch;
  const bool mine = c < a.C;
  float A[PER], S[PER], total = 0.f;
  float* kept = seg_state + (((size_t)b * a.nseg + seg) * a.C + min(c, a.C - 1)) * a.n;
  float* cell = state + ((size_t)max(slot, 0) * a.C + min(c, a.C - 1)) * a.n;
#pragma unroll
  for (int i = 0; i < PER; ++i) {
    const int n = part * PER + i;
    const bool on = mine && n < a.n;
    A[i] = on ? -__expf(ld(a_log + (size_t)c * a.n + n)) * LOG2E : 0.f;
    S[i] = 0.f;
    if (PASS == WHOLE && on && first > 0 && len > 0) S[i] = cell[n];
    if (PASS == OUTPUTS && on) S[i] = kept[n];
  }
  // this thread's share of a tile: tokens tt + j * 256 / CH of channel tc
  const int tc = tid % CH, tt = tid / CH, cc = min(c0 + tc, a.C - 1);
  const float bias = ld(dt_bias + cc), D = ld(skip + cc);
  const size_t tok0 = (size_t)b * a.S;
  T rx[PT], rp[PT], rz[PT], rb[PB];
  auto fetch = [&](int t0) {
#pragma unroll
    for (int j = 0; j < PT; ++j) {
      const size_t t = tok0 + min(t0 + tt + j * (256 / CH), len - 1);
      rx[j] = x[t * a.C + cc];
      rp[j] = pre[t * a.C + cc];
      if (PASS != STATES) rz[j] = z[t * a.zN + a.z_at + cc];
    }
#pragma unroll
    for (int j = 0; j < PB; ++j) {
      const int i = tid + j * 256, which = i / (TT * NP), t = i / NP % TT, n = i % NP;
      if (which < (PASS == STATES ? 1 : 2)) rb[j] = n < a.n ? bc[(tok0 + min(t0 + t, len - 1)) * a.bN + (which ? a.c_at : a.b_at) + n] : (T)0;
    }
  };
  if (len > lo) fetch(lo);
  for (int t0 = lo; t0 < len; t0 += TT) {
    float xv[PT], zv[PT];
#pragma unroll
    for (int j = 0; j < PT; ++j) {
      xv[j] = ld(rx + j);
      zv[j] = PASS == STATES ? 0.f : ld(rz + j);
      // tokens past the end leave the state as it is
      const float dt = t0 + tt + j * (256 / CH) < len ? softplusf(ld(rp + j) + bias) : 0.f;
      sd[tt + j * (256 / CH)][tc] = make_float2(dt, dt * xv[j]);
    }
#pragma unroll
    for (int j = 0; j < PB; ++j) {
      const int i = tid + j * 256;
      if (i < (PASS == STATES ? 1 : 2) * TT * NP) (&sb[0][0][0])[i] = ld(rb + j);
    }
    __syncthreads();
    if (t0 + TT < len) fetch(t0 + TT);
    const int n = min(TT, len - t0);
#pragma unroll 4
    for (int t = 0; t < TT; ++t) {
      const float2 d = sd[t][ch];
      float y = 0.f;
#pragma unroll
      for (int i = 0; i < PER; ++i) {
        S[i] = __builtin_amdgcn_exp2f(d.x * A[i]) * S[i] + d.y * sb[0][t][part * PER + i];
        if (PASS != STATES) y += S[i] * sb[1][t][part * PER + i];
      }
      if (PASS == STATES) total += d.x;
      else {
        y = lanes_sum<L>(y);
        if (part == 0) sy[t][ch] = y;
      }
    }
    __syncthreads();
    if (PASS == STATES) continue;
#pragma unroll
    for (int j = 0; j < PT; ++j) {
      const int t = tt + j * (256 / CH);
      if (t < n && c0 + tc < a.C)
        st(out + (tok0 + t0 + t) * a.K + a.out_at + c0 + tc, (sy[t][tc] + D * xv[j]) * siluf(zv[j]) * a.out_scale);
    }
  }
  // a row's own last segment leaves the state behind
  float* dst = PASS == STATES ? kept : row_len > lo && row_len <= lo + a.seg ? cell : nullptr;
  if (dst)
#pragma unroll
    for (int i = 0; i < PER; ++i)
      if (mine && part * PER + i < a.n) dst[part * PER + i] = S[i];
  if (PASS == STATES) {
    if (mine && part == 0) seg_dt[((size_t)b * a.nseg + seg) * a.C + c] = total;
    return;
  }
  for (int t = max(len, lo) + tt; t < min(a.S, lo + a.seg); t += 256 / CH)  // padding
    if (c0 + tc < a.C) st(out + (tok0 + t) * a.K + a.out_at + c0 + tc, 0.f);
}

// Final states of the segments (each from zero) -> the states they start from.
template <typename T>
__global__ __launch_bounds__(256) void segment_states_kernel(
    const T* __restrict__ a_log, const float* __restrict__ state, float* __restrict__ seg_state,
    const float* __restrict__ seg_dt, ScanArgs a, Step step) {
  const int i = blockIdx.x * 256 + threadIdx.x, b = blockIdx.y, slot = step.slot(b);
  const size_t cells = (size_t)a.C * a.n;
  if (i >= cells) return;
  const float A = -__expf(ld(a_log + i)) * LOG2E;
  float S = slot >= 0 && step.start > 0 ? state[(size_t)slot * cells + i] : 0.f;
  for (int s = 0; s < a.nseg; ++s) {
    float* p = seg_state + ((size_t)b * a.nseg + s) * cells + i;
    const float own = *p;
    *p = S;
    S = __builtin_amdgcn_exp2f(A * seg_dt[((size_t)b * a.nseg + s) * a.C + i / a.n]) * S + own;
  }
}

// Decode: one token a row; L lanes share a channel, PER states each.
template <typename T, int L, int PER>
__global__ __launch_bounds__(256) void scan_step_kernel(
    const T* __restrict__ x, const T* __restrict__ pre, const T* __restrict__ bc, const T* __restrict__ z,
    const T* __restrict__ a_log, const T* __restrict__ dt_bias, const T* __restrict__ skip, float* __restrict__ state,
    T* __restrict__ out, ScanArgs a, Step step) {
  const int c = blockIdx.x * (256 / L) + threadIdx.x / L, part = threadIdx.x % L, b = blockIdx.y;
  const int slot = step.slot(b);
  if (c >= a.C) return;
  T* dst = out + (size_t)b * a.K + a.out_at + c;
  if (slot < 0) {
    if (part == 0) st(dst, 0.f);
    return;
  }
  const bool fresh = step.first(b) == 0, vec = PER % 4 == 0 && a.n % 4 == 0;
  float* cell = state + ((size_t)slot * a.C + c) * a.n;
  float S[PER], al[PER];
#pragma unroll
  for (int i = 0; i < PER; i += 4) {
    const int n = part * PER + i;
    if (vec && n < a.n) {
      ld4(cell + n, S + i);
      ldv<4>(a_log + (size_t)c * a.n + n, al + i);
    } else {
#pragma unroll
      for (int j = 0; j < 4; ++j)
        if (i + j < PER) {
          S[i + j] = n + j < a.n ? cell[n + j] : 0.f;
          al[i + j] = n + j < a.n ? ld(a_log + (size_t)c * a.n + n + j) : 0.f;
        }
    }
  }
  const float xv = ld(x + (size_t)b * a.C + c), dt = softplusf(ld(pre + (size_t)b * a.C + c) + ld(dt_bias + c));
  const T* row = bc + (size_t)b * a.bN;
  float y = 0.f, Bv[PER], Cv[PER];
  const bool vec_bc = vec && ((a.bN | a.b_at | a.c_at) & 3) == 0;
#pragma unroll
  for (int i = 0; i < PER; i += 4) {
    const int n = part * PER + i;
    if (vec_bc && n < a.n) {
      ldv<4>(row + a.b_at + n, Bv + i);
      ldv<4>(row + a.c_at + n, Cv + i);
    } else {
#pragma unroll
      for (int j = 0; j < 4; ++j)
        if (i + j < PER) {
          Bv[i + j] = n + j < a.n ? ld(row + a.b_at + n + j) : 0.f;
          Cv[i + j] = n + j < a.n ? ld(row + a.c_at + n + j) : 0.f;
        }
    }
  }
#pragma unroll
  for (int i = 0; i < PER; ++i) {
    const int n = part * PER + i;
    if (n < a.n) {
      const float keep = fresh ? 0.f : __builtin_amdgcn_exp2f(dt * (-__expf(al[i]) * LOG2E)) * S[i];
      S[i] = keep + dt * xv * Bv[i];
      y += S[i] * Cv[i];
    }
  }
#pragma unroll
  for (int i = 0; i < PER; i += 4) {
    const int n = part * PER + i;
    if (vec && n < a.n) st4(cell + n, S + i);
    else
#pragma unroll
      for (int j = 0; j < 4; ++j)
        if (i + j < PER && n + j < a.n) cell[n + j] = S[i + j];
  }
  y = lanes_sum<L>(y);
  if (part == 0)
    st(dst, (y + ld(skip + c) * xv) * siluf(ld(z + (size_t)b * a.zN + a.z_at + c)) * a.out_scale);
}

// ===========================================================================
// host side
// ===========================================================================

// x: C columns of proj [B,S,N] from column `at` on
Tensor short_conv(Tensor proj, int64_t at, Tensor w, OptT bias, OptT in_bias, bool silu, Tensor ring, OptT slots,
                  OptT positions, OptT lens, int64_t start, bool decode, bool add) {
  const auto dt = io_type(proj);
  for (const Tensor& t : {w, ring}) check_io(t, dt);
  if (bias) { check_io(*bias, dt); CHK(bias->numel() == w.size(0)); }
  CHK(proj.dim() == 3 && w.dim() == 2 && ring.dim() == 3);
  const int B = proj.size(0), S = proj.size(1), N = proj.size(2), C = w.size(0), taps = w.size(1);
  CHK(at + C <= N && taps >= 1 && ring.size(1) == taps && ring.size(2) == C);
  CHK((slots || B <= ring.size(0)) && (!decode || S == 1) && B <= 65535);
  auto out = torch::empty({B, S, C}, proj.options());
  if (B == 0 || S == 0) return out;
  const Step step = make_step(slots, positions, lens, start, decode, B);
  if (in_bias) { check_io(*in_bias, dt); CHK(in_bias->numel() == C); }
  const ConvArgs a{S, C, N, (int)at, taps, silu, add};
  const hipStream_t stream = cur_stream();
  const bool vec = ((C | N | (int)at) & 3) == 0;
  CHK((S + RUN - 1) / RUN <= 65535);
  const dim3 grid((C + (vec ? 1023 : 255)) / (vec ? 1024 : 256), (S + RUN - 1) / RUN, B);
#define CONV(V, TAPS)                                                                                            \
  hipLaunchKernelGGL((short_conv_kernel<T, V, TAPS>), grid, dim3(256), 0, stream, P<T>(proj), P<T>(w),             \
                     bias ? P<T>(*bias) : nullptr, in_bias ? P<T>(*in_bias) : nullptr, M<T>(ring), M<T>(out), a, step)
#define CONV_TAPS(V)               \
  if (taps == 4) CONV(V, 4);       \
  else if (taps == 3) CONV(V, 3);  \
  else if (taps == 2) CONV(V, 2);  \
  else CONV(V, 0)
  BY_TYPE(dt, {
    if (vec) { CONV_TAPS(4); } else { CONV_TAPS(1); }
    if (!decode)
      hipLaunchKernelGGL((keep_inputs_kernel<T>), dim3(std::min(taps, S), B), dim3(256), 0, stream, P<T>(proj), M<T>(ring), a, step);
  });
#undef CONV_TAPS
#undef CONV
  return out;
}

// x, pre [B,S,C]; bc [B,S,*] with B and C at columns b_at and c_at; the gate
// is C columns of z [B,S,*]; a_log [C,n]; state [slots,C,n]
void selective_scan(Tensor x, Tensor pre, Tensor bc, int64_t b_at, int64_t c_at, Tensor z, int64_t z_at, Tensor a_log,
                    Tensor dt_bias, Tensor skip, Tensor state, OptT slots, OptT positions, OptT lens, int64_t start,
                    bool decode, Tensor out, int64_t out_at, double out_scale) {
  const auto dt = io_type(x);
  for (const Tensor& t : {pre, bc, z, a_log, dt_bias, skip, out}) check_io(t, dt);
  check_io(state, torch::kFloat32);
  CHK(x.dim() == 3 && x.sizes() == pre.sizes() && bc.dim() == 3 && z.dim() == 3 && out.dim() == 3 && a_log.dim() == 2);
  const int B = x.size(0), S = x.size(1), C = x.size(2), n = a_log.size(1);
  for (const Tensor& t : {bc, z, out}) CHK(t.size(0) == B && t.size(1) == S);
  CHK(a_log.size(0) == C && dt_bias.numel() == C && skip.numel() == C && n >= 1);
  CHK(b_at + n <= bc.size(2) && c_at + n <= bc.size(2) && z_at + C <= z.size(2) && out_at + C <= out.size(2));
  CHK(state.dim() == 3 && state.size(1) == C && state.size(2) == n && (slots || B <= state.size(0)) && (!decode || S == 1));
  TORCH_CHECK(n <= 256, "a state of ", n, " numbers per channel (at most 256)");
  if (B == 0 || S == 0) return;
  CHK(B <= 65535);
  const Step step = make_step(slots, positions, lens, start, decode, B);
  ScanArgs a{S, C, n, (int)z.size(2), (int)z_at, (int)bc.size(2), (int)b_at, (int)c_at, (int)out.size(2),
                   (int)out_at, (float)out_scale, S, 1};
  const hipStream_t stream = cur_stream();
  // blocks of the form that does the least work per state; if they do not fill
  // the chip, long rows are cut into segments and short ones take more lanes
  const int lanes = n <= 32 ? 4 : 16, blocks = (C + 256 / lanes - 1) / (256 / lanes) * B;
  if (!decode && blocks < 256) {
    a.nseg = std::max(1, std::min(S / 64, (512 + blocks - 1) / blocks));
    a.seg = ((S + a.nseg - 1) / a.nseg + 15) / 16 * 16;
    a.nseg = (S + a.seg - 1) / a.seg;
  }
  const bool wide = !decode && blocks < 256 && a.nseg == 1;
  Tensor seg_state, seg_dt;
  if (a.nseg > 1) {
    seg_state = f32(x, {B, a.nseg, C, n});
    seg_dt = f32(x, {B, a.nseg, C});
  }
  float *ss = a.nseg > 1 ? M<float>(seg_state) : nullptr, *sd = a.nseg > 1 ? M<float>(seg_dt) : nullptr;
#define STEP(L, PER)                                                                                                   \
  hipLaunchKernelGGL((scan_step_kernel<T, L, PER>), dim3((C + 256 / L - 1) / (256 / L), B), dim3(256), 0, stream, P<T>(x), \
                     P<T>(pre), P<T>(bc), P<T>(z), P<T>(a_log), P<T>(dt_bias), P<T>(skip), M<float>(state), M<T>(out), a, step)
#define PASS(L, PER, WHICH)                                                                                            \
  hipLaunchKernelGGL((scan_kernel<T, L, PER, WHICH>), dim3((C + 256 / L - 1) / (256 / L), B, a.nseg), dim3(256), 0,    \
                     stream, P<T>(x), P<T>(pre), P<T>(bc), P<T>(z), P<T>(a_log), P<T>(dt_bias), P<T>(skip),            \
                     M<float>(state), ss, sd, M<T>(out), a, step)
#define SCAN(L, PER)                                                                                              \
  if (a.nseg == 1) PASS(L, PER, WHOLE);                                                                           \
  else {                                                                                                          \
    PASS(L, PER, STATES);                                                                                         \
    hipLaunchKernelGGL((segment_states_kernel<T>), dim3((C * n + 255) / 256, B), dim3(256), 0, stream, P<T>(a_log), \
                       P<float>(state), ss, sd, a, step);                                                         \
    PASS(L, PER, OUTPUTS);                                                                                        \
  }
  BY_TYPE(dt, {
    if (decode) {
      if (n <= 16) STEP(4, 4);
      else if (n <= 32) STEP(4, 8);
      else if (n <= 64) STEP(16, 4);
      else if (n <= 128) STEP(16, 8);
      else STEP(16, 16);
    } else if (n <= 16) {
      if (wide) PASS(16, 1, WHOLE);
      else { SCAN(4, 4) }
    } else if (n <= 32) {
      if (wide) PASS(16, 2, WHOLE);
      else { SCAN(4, 8) }
    } else if (n <= 64) { SCAN(16, 4) }
    else if (n <= 128) { SCAN(16, 8) }
    else { SCAN(16, 16) }
  });
#undef SCAN
#undef PASS
#undef STEP
}

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.def("short_conv", &short_conv, "short causal convolution with bias, and silu; added to its input",
        py::arg("proj"), py::arg("at"), py::arg("w"), py::arg("bias"), py::arg("in_bias"), py::arg("silu"),
        py::arg("ring"), py::arg("slots"), py::arg("positions"), py::arg("lens"), py::arg("start"), py::arg("decode"),
        py::arg("add") = false);
  m.def("selective_scan", &selective_scan, "selective state space scan with skip and gate");
}
