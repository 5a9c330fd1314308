// CDNA4 (gfx950) kernels of the token mixers in models/mixers.py, and of the
// norms around an fp32 residual stream:
//   - sandwich norm: stream += norm(sublayer output), then the stream's norm
//     for the next sublayer, one pass
//   - gated delta rule and WKV recurrences: for prompts the factors of
//     16-token chunks (short convolutions, unit norms, decays) and a scan over
//     chunks on fp32 MFMA, one fused kernel per decode step
//
// Two element types, bf16 and fp32. Recurrent state, norms and everything that
// feeds a recurrence after its projections are fp32 in both.
//
// Rows of a step address state by slot (struct Step): slot -1 is a parked row,
// which reads and writes no state and yields zeros. A row at position 0
// ignores what its slot holds.

#include "common.h"

// ---------------------------------------------------------------------------
// norms around the fp32 stream
// ---------------------------------------------------------------------------

// y null: h = norm(x; w_next) only. With `rows`, a row of y is the weighted sum
// of `top` of its rows. copy: h is the stream as it is. One block per row; the
// row stays in registers (NC chunks of 256*V elements).
template <typename T, int V, int NC>
__global__ __launch_bounds__(256) void sandwich_norm_kernel(
    const T* __restrict__ y, const int* __restrict__ rows, const float* __restrict__ weight, int top, int ys,
    float* __restrict__ x, const T* __restrict__ w_post, const T* __restrict__ w_next, T* __restrict__ h, int copy,
    int D, float eps) {
  const size_t off = (size_t)blockIdx.x * D;
  __shared__ float red[8];
  float xv[NC * V];
#pragma unroll
  for (int c = 0; c < NC; ++c) {
    const int i = (c * 256 + threadIdx.x) * V;
    if (i < D) ldv<V>(x + off + i, xv + c * V);
    else
#pragma unroll
      for (int j = 0; j < V; ++j) xv[c * V + j] = 0.f;
  }
  if (y) {
    float yv[NC * V], acc = 0.f;
#pragma unroll
    for (int c = 0; c < NC; ++c) {
      const int i = (c * 256 + threadIdx.x) * V;
      if (i < D) {
        if (!rows) ldv<V>(y + (size_t)blockIdx.x * ys + i, yv + c * V);
        else
#pragma unroll
          for (int j = 0; j < V; ++j) yv[c * V + j] = 0.f;
        for (int k = 0; rows && k < top; ++k) {
          const float wk = weight ? weight[(size_t)blockIdx.x * top + k] : 1.f;
          float v[V];
          ldv<V>(y + (size_t)rows[(size_t)blockIdx.x * top + k] * ys + i, v);
#pragma unroll
          for (int j = 0; j < V; ++j) yv[c * V + j] += wk * v[j];
        }
#pragma unroll
        for (int j = 0; j < V; ++j) acc += yv[c * V + j] * yv[c * V + j];
      }
    }
    const float inv = 1.f / sqrtf(block_sum(acc, red) / (float)D + eps);
#pragma unroll
    for (int c = 0; c < NC; ++c) {
      const int i = (c * 256 + threadIdx.x) * V;
      if (i < D) {
        float w[V];
        ldv<V>(w_post + i, w);
#pragma unroll
        for (int j = 0; j < V; ++j) xv[c * V + j] += yv[c * V + j] * inv * (1.f + w[j]);
        stv<V>(x + off + i, xv + c * V);
        if (copy) stv<V>(h + off + i, xv + c * V);
      }
    }
  }
  if (!w_next) return;
  float acc = 0.f;
#pragma unroll
  for (int i = 0; i < NC * V; ++i) acc += xv[i] * xv[i];
  const float inv = 1.f / sqrtf(block_sum(acc, red + 4) / (float)D + eps);
#pragma unroll
  for (int c = 0; c < NC; ++c) {
    const int i = (c * 256 + threadIdx.x) * V;
    if (i < D) {
      float w[V], o[V];
      ldv<V>(w_next + i, w);
#pragma unroll
      for (int j = 0; j < V; ++j) o[j] = xv[c * V + j] * inv * (1.f + w[j]);
      stv<V>(h + off + i, o);
    }
  }
}

// ---------------------------------------------------------------------------
// elementwise
// ---------------------------------------------------------------------------

template <typename T, int V>
__global__ __launch_bounds__(256) void swiglu_kernel(const T* __restrict__ gu, T* __restrict__ out, long long n, int I) {
  const long long i = ((long long)blockIdx.x * 256 + threadIdx.x) * V;
  if (i >= n) return;
  const long long row = i / I;
  const int c = (int)(i - row * I);
  float g[V], u[V];
  ldv<V>(gu + row * 2 * I + c, g);
  ldv<V>(gu + row * 2 * I + I + c, u);
#pragma unroll
  for (int j = 0; j < V; ++j) u[j] *= siluf(g[j]);
  stv<V>(out + i, u);
}

template <typename T>
__global__ __launch_bounds__(256) void tanh_kernel(const T* __restrict__ x, T* __restrict__ out, long long n) {
  const long long i = (long long)blockIdx.x * 256 + threadIdx.x;
  if (i < n) st(out + i, tanhf(ld(x + i)));
}

// ---------------------------------------------------------------------------
// recurrences
// ---------------------------------------------------------------------------

// Last inputs of a chunk into a ring of rows by position (convolutions,
// token shift). Up to three column ranges of src, side by side in the ring.
struct Columns { int at[3], n[3]; };

template <typename T>
__global__ __launch_bounds__(256) void remember_kernel(
    const T* __restrict__ src, T* __restrict__ ring, int S, int N, int M, int C, Columns cols, Step step) {
  const int b = blockIdx.y, slot = step.slot(b), len = step.len(b, S);
  const int s = len - 1 - blockIdx.x;
  if (slot < 0 || s < 0) return;
  const T* row = src + ((size_t)b * S + s) * N;
  T* dst = ring + ((size_t)slot * M + (step.first(b) + s) % M) * C;
  for (int i = threadIdx.x; i < C; i += 256) {
    int c = i, r = 0;
    while (r < 2 && c >= cols.n[r]) c -= cols.n[r++];
    dst[i] = row[cols.at[r] + c];
  }
}

struct RecArgs {
  int S, H, G, N, K;
  int dim, vdim, dp, taps;               // dp: padded key channels
  int q_at, k_at, v_at, b_at, out_at;
  float eps, out_scale;
};

// sum over taps of a channel's inputs, then silu; ch: channel in the ring
template <typename T>
DEVINL float conv_silu(const T* proj, const T* ring, const T* taps_w, int s, int first, int col, int ch, int wch,
                       int C, const RecArgs& a) {
  float y = 0.f;
  for (int j = 0; j < a.taps; ++j) {
    const int back = a.taps - 1 - j;
    float x = 0.f;
    if (s >= back) x = ld(proj + (long long)(s - back) * a.N + col);
    else if (first + s >= back) x = ld(ring + (size_t)((first + s - back) % a.taps) * C + ch);
    y += x * ld(taps_w + wch * a.taps + j);
  }
  return siluf(y);
}

// PER consecutive channels of a lane, those past n as zero; `vec`: the
// address allows one load
template <int PER, typename T>
DEVINL void ld_lane(const T* p, int c, int n, bool vec, float* o) {
  if (PER == 4 && vec && c + 3 < n) { ld4(p + c, o); return; }
  if (PER == 2 && vec && c + 1 < n) { ld2(p + c, o); return; }
#pragma unroll
  for (int i = 0; i < PER; ++i) o[i] = c + i < n ? ld(p + c + i) : 0.f;
}
template <int PER, typename T>
DEVINL void st_lane(T* p, int c, int n, bool vec, const float* o) {
  if (PER == 4 && vec && c + 3 < n) { st4(p + c, o); return; }
  if (PER == 2 && vec && c + 1 < n) { st2(p + c, o); return; }
#pragma unroll
  for (int i = 0; i < PER; ++i)
    if (c + i < n) st(p + c + i, o[i]);
}

// A lane's channels through a causal convolution and silu, token by token:
// weights and the last inputs stay in registers. TAPS 0: any number of taps,
// inputs read again for every token.
template <typename T, int TAPS, int PER>
struct Conv {
  static constexpr int NT = TAPS ? TAPS : 1;
  float w[NT][PER], x[NT][PER];
  const T *rows, *ring, *tw;
  int col, ch, c, n, first;
  bool vec;
  DEVINL void history(int t, float* o, int C, const RecArgs& a) const {  // input of chunk token t (t < 0: before it)
    if (t >= 0) ld_lane<PER>(rows + (long long)t * a.N + col, c, n, vec, o);
    else if (first + t >= 0) ld_lane<PER>(ring + (size_t)((first + t) % a.taps) * C + ch, c, n, false, o);
    else
#pragma unroll
      for (int i = 0; i < PER; ++i) o[i] = 0.f;
  }
  DEVINL void begin(int s0, int C, const RecArgs& a) {
    if (!TAPS) return;
#pragma unroll
    for (int i = 0; i < PER; ++i)
#pragma unroll
      for (int j = 0; j < NT; ++j) w[j][i] = c + i < n ? ld(tw + (size_t)(c + i) * TAPS + j) : 0.f;
#pragma unroll
    for (int j = 1; j < NT; ++j) history(s0 - NT + j, x[j], C, a);
  }
  DEVINL void next(int s, int C, const RecArgs& a, float* y) {
#pragma unroll
    for (int i = 0; i < PER; ++i) y[i] = 0.f;
    if (!TAPS) {
      for (int j = 0; j < a.taps; ++j) {
        float v[PER];
        history(s - (a.taps - 1 - j), v, C, a);
#pragma unroll
        for (int i = 0; i < PER; ++i) y[i] += v[i] * (c + i < n ? ld(tw + (size_t)(c + i) * a.taps + j) : 0.f);
      }
    } else {
#pragma unroll
      for (int j = 0; j + 1 < NT; ++j)
#pragma unroll
        for (int i = 0; i < PER; ++i) x[j][i] = x[j + 1][i];
      history(s, x[NT - 1], C, a);
#pragma unroll
      for (int j = 0; j < NT; ++j)
#pragma unroll
        for (int i = 0; i < PER; ++i) y[i] += x[j][i] * w[j][i];
    }
#pragma unroll
    for (int i = 0; i < PER; ++i) y[i] = siluf(y[i]);
  }
};

// --- prompts, 16 tokens (a chunk) at a time -------------------------------
// With L_t the log decays summed up to token t of a chunk and S the state
// before it, the delta rule's 16 sequential updates are
//   U = T (V - K~ S),  O = Q~ S + B U,  S' = e^{L_15} S + K^T U
//   K~_t = k_t e^{L_t}   Q~_t = q_t e^{L_t}   K^_s = k_s e^{L_15 - L_s}
//   A_ts = sum_d k_t k_s e^{L_t - L_s} (s < t),  B_ts = the same with q_t (s <= t)
//   T = (I + diag(beta) A)^-1 diag(beta)
// and WKV's, which read before they write, the same with U = V,
// Q~_t = r_t e^{L_(t-1)}, B_ts = sum_d r_t k_s e^{L_(t-1) - L_s} (s < t) and
// B_tt the bonus. Every exponent is <= 0, so nothing overflows however strong
// the decays are. chunk_prep_kernel makes the factors of all chunks in
// parallel, chunk_scan_kernel walks the chunks with fp32 MFMA.
//
// Factors of a (row, chunk, head), in floats: Q~ [16][dp] | K^ transposed
// [dp][16] | e^{L_15} [dp] | B [16][16] | T [16][16] | K~ [16][dp] (the last
// two only for the delta rule).
constexpr int CHUNK = 16;
DEVINL int chunk_floats(bool delta, int dp) { return delta ? 49 * dp + 512 : 33 * dp + 256; }

// One block per (head, chunk, row). DELTA: x0 is the fused projection, x1 and
// x2 unused; c0..c2 the taps of q, k, v; d0 = A_log, d1 = dt_bias. WKV: x0..x2
// are r, k, v; d0 = w0, d1 = u.
template <typename T, bool DELTA, int TAPS, int PER>
__global__ __launch_bounds__(256) void chunk_prep_kernel(
    const T* __restrict__ x0, const T* __restrict__ x1, const T* __restrict__ x2, const T* __restrict__ c0,
    const T* __restrict__ c1, const T* __restrict__ c2, const T* __restrict__ pre, const T* __restrict__ d0,
    const T* __restrict__ d1, const T* __restrict__ ring, float* __restrict__ factors, float* __restrict__ v,
    int chunks, RecArgs a, Step step) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const int dps = a.dp + 4;
  float *sq = lds, *sk = sq + CHUNK * dps, *sl = sk + CHUNK * dps;
  float *sA = sl + CHUNK * dps, *sB = sA + 256, *sb = sB + 256;  // sb: beta or bonus per token
  const int h = blockIdx.x, b = blockIdx.z, tid = threadIdx.x, g = h / (a.H / a.G);
  const int slot = step.slot(b), len = step.len(b, a.S), s0 = blockIdx.y * CHUNK;
  if (slot < 0 || s0 >= len) return;
  const int c = (tid & 63) * PER, t0 = (tid >> 6) * 4;  // a wave takes 4 tokens
  float* out = factors + (((size_t)b * chunks + blockIdx.y) * a.H + h) * chunk_floats(DELTA, a.dp);
  float bias[PER];
  if (DELTA) {
    const int C = 2 * a.G * a.dim + a.H * a.vdim, first = step.first(b), kw = a.G * a.dim;
    const int qch = g * a.dim, vch = h * a.vdim;
    const T* rows = x0 + (size_t)b * a.S * a.N;
    const T* hist = ring + (size_t)slot * a.taps * C;
    const bool vd = ((a.dim | a.N | a.q_at | a.k_at) & 3) == 0, ve = ((a.vdim | a.N | a.v_at) & 3) == 0;
    Conv<T, TAPS, PER> cq{{}, {}, rows, hist, c0 + (size_t)qch * a.taps, a.q_at + qch, qch, c, a.dim, first, vd};
    Conv<T, TAPS, PER> ck{{}, {}, rows, hist, c1 + (size_t)qch * a.taps, a.k_at + qch, kw + qch, c, a.dim, first, vd};
    Conv<T, TAPS, PER> cv{{}, {}, rows, hist, c2 + (size_t)vch * a.taps, a.v_at + vch, 2 * kw + vch, c, a.vdim, first, ve};
    const bool any = s0 + t0 < len;
    if (any) {
      cq.begin(s0 + t0, C, a);
      ck.begin(s0 + t0, C, a);
      cv.begin(s0 + t0, C, a);
    }
    const float A = __expf(ld(d0 + h)), qscale = 1.f / sqrtf((float)a.dim);
    ld_lane<PER>(d1 + (size_t)h * a.dim, c, a.dim, (a.dim & 3) == 0, bias);
    for (int t = t0; t < t0 + 4; ++t) {
      const int s = s0 + t;
      float q[PER], k[PER], y[PER], lg[PER], beta = 0.f;
#pragma unroll
      for (int i = 0; i < PER; ++i) q[i] = k[i] = lg[i] = 0.f;
      if (s < len) {
        const size_t head = ((size_t)b * a.S + s) * a.H + h;
        cq.next(s, C, a, q);
        ck.next(s, C, a, k);
        cv.next(s, C, a, y);
        st_lane<PER>(v + head * a.vdim, c, a.vdim, (a.vdim & 3) == 0, y);
        float qq = 0.f, kk = 0.f;
#pragma unroll
        for (int i = 0; i < PER; ++i) {
          qq += q[i] * q[i];
          kk += k[i] * k[i];
        }
        const float qi = qscale / sqrtf(wave_sum(qq) + 1e-6f), ki = 1.f / sqrtf(wave_sum(kk) + 1e-6f);
        ld_lane<PER>(pre + head * a.dim, c, a.dim, (a.dim & 3) == 0, lg);
#pragma unroll
        for (int i = 0; i < PER; ++i) {
          q[i] *= qi;
          k[i] *= ki;
          lg[i] = c + i < a.dim ? -A * softplusf(lg[i] + bias[i]) : 0.f;
        }
        beta = sigmoidf(ld(rows + (size_t)s * a.N + a.b_at + h));
      }
      st_lane<PER>(sq + t * dps, c, a.dp, true, q);
      st_lane<PER>(sk + t * dps, c, a.dp, true, k);
      st_lane<PER>(sl + t * dps, c, a.dp, true, lg);
      if (c == 0) sb[t] = beta;
    }
  } else {
    const bool vec = (a.dim & 3) == 0;
    float u[PER];
    ld_lane<PER>(d0 + (size_t)h * a.dim, c, a.dim, vec, bias);
    ld_lane<PER>(d1 + (size_t)h * a.dim, c, a.dim, vec, u);
#pragma unroll
    for (int t = t0; t < t0 + 4; ++t) {
      const int s = s0 + t;
      float q[PER], k[PER], y[PER], lg[PER], bonus = 0.f;
#pragma unroll
      for (int i = 0; i < PER; ++i) q[i] = k[i] = lg[i] = 0.f;
      if (s < len) {
        const size_t src = (((size_t)b * a.S + s) * a.H + h) * a.dim;
        ld_lane<PER>(x0 + src, c, a.dim, vec, q);
        ld_lane<PER>(x1 + src, c, a.dim, vec, k);
        ld_lane<PER>(x2 + src, c, a.dim, vec, y);
        ld_lane<PER>(pre + src, c, a.dim, vec, lg);
        st_lane<PER>(v + src, c, a.dim, vec, y);
#pragma unroll
        for (int i = 0; i < PER; ++i) {
          lg[i] = c + i < a.dim ? -__expf(lg[i] + bias[i]) : 0.f;
          bonus += q[i] * k[i] * u[i];
        }
      }
      bonus = wave_sum(bonus);
      st_lane<PER>(sq + t * dps, c, a.dp, true, q);
      st_lane<PER>(sk + t * dps, c, a.dp, true, k);
      st_lane<PER>(sl + t * dps, c, a.dp, true, lg);
      if (c == 0) sb[t] = bonus;
    }
  }
  __syncthreads();
  for (int d = tid; d < a.dp; d += 256) {
    float run = 0.f;
#pragma unroll
    for (int t = 0; t < CHUNK; ++t) {
      run += sl[t * dps + d];
      sl[t * dps + d] = run;
    }
    out[32 * a.dp + d] = __expf(run);
  }
  __syncthreads();
  if (tid < 136) {  // pairs s <= t
    int t = (int)((sqrtf(8.f * tid + 1.f) - 1.f) * .5f);
    if ((t + 1) * (t + 2) / 2 <= tid) ++t;
    if (t * (t + 1) / 2 > tid) --t;
    const int s = tid - t * (t + 1) / 2;
    float A = 0.f, B = 0.f;
    if (DELTA || s < t) {
      const float *kt = sk + t * dps, *ks = sk + s * dps, *qt = sq + t * dps;
      const float *lt = sl + (DELTA ? t : t - 1) * dps, *ls = sl + s * dps;
      for (int d = 0; d < a.dp; d += 4) {
        float xt[4], xs[4], xq[4], et[4], es[4];
        ld4(ks + d, xs);
        ld4(qt + d, xq);
        ld4(lt + d, et);
        ld4(ls + d, es);
        if (DELTA) ld4(kt + d, xt);
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const float w = xs[i] * __expf(et[i] - es[i]);
          if (DELTA) A += xt[i] * w;
          B += xq[i] * w;
        }
      }
    } else {
      B = sb[t];
    }
    sA[t * 16 + s] = A;
    sB[t * 16 + s] = B;
  } else {
    int p = tid - 136, s = 1;  // pairs s > t
    while (p >= s) p -= s++;
    sA[p * 16 + s] = 0.f;
    sB[p * 16 + s] = 0.f;
  }
  const int row4 = a.dp >> 2;
  for (int e = tid; e < CHUNK * row4; e += 256) {
    const int t = e / row4, d = (e - t * row4) * 4;
    float q[4], l[4] = {0.f, 0.f, 0.f, 0.f};
    ld4(sq + t * dps + d, q);
    if (DELTA || t > 0) ld4(sl + (DELTA ? t : t - 1) * dps + d, l);
    if (DELTA) {
      float k[4];
      ld4(sk + t * dps + d, k);
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        l[i] = __expf(l[i]);
        k[i] *= l[i];
        q[i] *= l[i];
      }
      st4(out + 33 * a.dp + 512 + t * a.dp + d, k);
    } else {
#pragma unroll
      for (int i = 0; i < 4; ++i) q[i] *= __expf(l[i]);
    }
    st4(out + t * a.dp + d, q);
  }
  for (int e = tid; e < a.dp * 4; e += 256) {
    const int d = e >> 2, t = (e & 3) * 4;
    const float end = sl[(CHUNK - 1) * dps + d];
    float k[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) k[i] = sk[(t + i) * dps + d] * __expf(end - sl[(t + i) * dps + d]);
    st4(out + 16 * a.dp + e * 4, k);
  }
  __syncthreads();
  out[33 * a.dp + tid] = sB[tid];
  if (DELTA && tid < CHUNK) {  // column tid of T by forward substitution
    float x[CHUNK];
#pragma unroll
    for (int t = 0; t < CHUNK; ++t) {
      float r = t == tid ? 1.f : 0.f;
#pragma unroll
      for (int s = 0; s < CHUNK; ++s)
        if (s < t) r -= sA[t * 16 + s] * x[s];
      x[t] = r * sb[t];
      out[33 * a.dp + 256 + t * 16 + tid] = x[t];
    }
  }
}

// A wave holds 16 columns of a head's state as MFMA accumulators (NI tiles of
// 16 key channels). A lane's accumulator element r of tile i is channel
// i*16 + quad*4 + r of its column, so the accumulators are at the same time
// the right-hand operands of the products with S: step (i, r) of an
// f32 16x16x4 MFMA contracts the four channels its quads hold.
// KS > 1: KS of a block's 4 waves share a column group, each holding its part
// of the channels, and add their partial products through LDS (more blocks and
// shorter chunks where there are few sequences).
template <bool DELTA, int NI, int KS>
__global__ __launch_bounds__(256) void chunk_scan_kernel(
    const float* __restrict__ factors, const float* __restrict__ v, float* __restrict__ state, float* __restrict__ o,
    int chunks, RecArgs a, Step step) {
  constexpr int DP = 16 * NI, QS = DP + 4, TS = 20;  // padded LDS rows: no bank conflicts
  constexpr int FLOATS = DELTA ? 49 * DP + 512 : 33 * DP + 256, NL = (FLOATS / 4 + 255) / 256;
  constexpr int NT = NI / KS;  // tiles of this wave
  constexpr int AT_KT = 16 * QS, AT_E = AT_KT + DP * TS, AT_B = AT_E + DP, AT_T = AT_B + 16 * TS, AT_K = AT_T + 16 * TS;
  __shared__ __attribute__((aligned(16))) float lds[DELTA ? AT_K + 16 * QS : AT_T];
  __shared__ floatx4 part_p[KS > 1 && DELTA ? 256 : 1], part_o[KS > 1 ? 256 : 1];
  const int h = blockIdx.y, b = blockIdx.z, tid = threadIdx.x;
  const int slot = step.slot(b), len = step.len(b, a.S);
  if (slot < 0) return;
  const int lane = tid & 63, m = lane & 15, quad = lane >> 4, ks = (tid >> 6) % KS;
  const int col = (blockIdx.x * (4 / KS) + (tid >> 6) / KS) * 16 + m, d0 = ks * NT * 16 + quad * 4;
  const bool mine = col < a.vdim;
  // where this thread's float4s of a chunk's factors go
  int dst[NL];
#pragma unroll
  for (int i = 0; i < NL; ++i) {
    int e = (tid + i * 256) * 4;
    if (e < 16 * DP) dst[i] = e / DP * QS + e % DP;
    else if (e < 32 * DP) { e -= 16 * DP; dst[i] = AT_KT + e / 16 * TS + e % 16; }
    else if (e < 33 * DP) dst[i] = AT_E + e - 32 * DP;
    else if (e < 33 * DP + 256) { e -= 33 * DP; dst[i] = AT_B + e / 16 * TS + e % 16; }
    else if (e < 33 * DP + 512) { e -= 33 * DP + 256; dst[i] = AT_T + e / 16 * TS + e % 16; }
    else { e -= 33 * DP + 512; dst[i] = AT_K + e / DP * QS + e % DP; }
  }
  floatx4 S[NT];
  float* base = state + (((size_t)slot * a.H + h) * a.vdim + (mine ? col : 0)) * DP + d0;
  const bool fresh = step.first(b) == 0;
#pragma unroll
  for (int i = 0; i < NT; ++i) S[i] = fresh || !mine ? (floatx4)(0.f) : *(const floatx4*)(base + i * 16);
  const size_t tok0 = (size_t)b * a.S, vstride = (size_t)a.H * a.vdim, vcol = (size_t)h * a.vdim + col;
  floatx4 rf[NL], rv;
  auto fetch = [&](int t0) {
    const float* src = factors + (((size_t)b * chunks + t0 / CHUNK) * a.H + h) * FLOATS;
#pragma unroll
    for (int i = 0; i < NL; ++i) {
      const int e = (tid + i * 256) * 4;
      if (e < FLOATS) rf[i] = *(const floatx4*)(src + e);
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int t = t0 + quad * 4 + r;
      rv[r] = mine && t < len ? v[(tok0 + t) * vstride + vcol] : 0.f;
    }
  };
  if (len > 0) fetch(0);
  for (int t0 = 0; t0 < len; t0 += CHUNK) {
    __syncthreads();  // everyone is done with the previous chunk's factors
#pragma unroll
    for (int i = 0; i < NL; ++i)
      if ((tid + i * 256) * 4 < FLOATS) *(floatx4*)(lds + dst[i]) = rf[i];
    const floatx4 V = rv;
    __syncthreads();
    if (t0 + CHUNK < len) fetch(t0 + CHUNK);
    floatx4 O = (floatx4)(0.f), P = (floatx4)(0.f);
#pragma unroll
    for (int i = 0; i < NT; ++i) {
      const floatx4 q4 = *(const floatx4*)(lds + m * QS + i * 16 + d0);
      floatx4 k4;
      if (DELTA) k4 = *(const floatx4*)(lds + AT_K + m * QS + i * 16 + d0);
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        if (DELTA) P = __builtin_amdgcn_mfma_f32_16x16x4f32(k4[r], S[i][r], P, 0, 0, 0);
        O = __builtin_amdgcn_mfma_f32_16x16x4f32(q4[r], S[i][r], O, 0, 0, 0);
      }
    }
    if (KS > 1) {
      if (DELTA) part_p[tid] = P;
      part_o[tid] = O;
      __syncthreads();
#pragma unroll
      for (int i = 1; i < KS; ++i) {
        const int other = tid + (((ks + i) % KS) - ks) * 64;
        if (DELTA) P += part_p[other];
        O += part_o[other];
      }
    }
    floatx4 U = V;
    if (DELTA) {
      const floatx4 W = V - P, t4 = *(const floatx4*)(lds + AT_T + m * TS + quad * 4);
      U = (floatx4)(0.f);
#pragma unroll
      for (int r = 0; r < 4; ++r) U = __builtin_amdgcn_mfma_f32_16x16x4f32(t4[r], W[r], U, 0, 0, 0);
    }
    const floatx4 b4 = *(const floatx4*)(lds + AT_B + m * TS + quad * 4);
#pragma unroll
    for (int r = 0; r < 4; ++r) O = __builtin_amdgcn_mfma_f32_16x16x4f32(b4[r], U[r], O, 0, 0, 0);
#pragma unroll
    for (int i = 0; i < NT; ++i) S[i] *= *(const floatx4*)(lds + AT_E + i * 16 + d0);
#pragma unroll
    for (int r = 0; r < 4; ++r)  // tiles innermost: consecutive MFMAs are independent
#pragma unroll
      for (int i = 0; i < NT; ++i)
        S[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(lds[AT_KT + ((ks * NT + i) * 16 + m) * TS + quad * 4 + r], U[r], S[i], 0, 0, 0);
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int t = t0 + quad * 4 + r;
      if (mine && ks == 0 && t < len) o[(tok0 + t) * vstride + vcol] = O[r];
    }
  }
  if (mine && len > 0)
#pragma unroll
    for (int i = 0; i < NT; ++i) *(floatx4*)(base + i * 16) = S[i];
}

// rows of the state that lane r (0..15) of a column holds: vectors of V
template <int RPL> struct Rows {
  static constexpr int V = RPL % 4 == 0 ? 4 : RPL % 2 == 0 ? 2 : 1;
  static DEVINL int at(int j, int r) { return j * 16 * V + V * r; }  // j < RPL / V
};
template <int RPL>
DEVINL void load_rows(const float* p, int r, float* o) {
#pragma unroll
  for (int j = 0; j < RPL / Rows<RPL>::V; ++j) ldv<Rows<RPL>::V>(p + Rows<RPL>::at(j, r), o + j * Rows<RPL>::V);
}
template <int RPL>
DEVINL void store_rows(float* p, int r, const float* o) {
#pragma unroll
  for (int j = 0; j < RPL / Rows<RPL>::V; ++j) stv<Rows<RPL>::V>(p + Rows<RPL>::at(j, r), o + j * Rows<RPL>::V);
}

// one token of a column; s: the column's rows in this lane. Returns the
// column's output (in all 16 lanes).
template <bool DELTA, int RPL>
DEVINL float rec_step(float* s, const float* q, const float* k, const float* g, float v, float beta, float dot) {
  float p1 = 0.f, p2 = 0.f;
  if (DELTA) {
#pragma unroll
    for (int i = 0; i < RPL; ++i) {
      s[i] *= g[i];
      p1 += s[i] * k[i];
      p2 += s[i] * q[i];
    }
    p1 = row_sum(p1);
    p2 = row_sum(p2);
    const float u = beta * (v - p1);
#pragma unroll
    for (int i = 0; i < RPL; ++i) s[i] += k[i] * u;
    return p2 + u * dot;
  }
#pragma unroll
  for (int i = 0; i < RPL; ++i) {
    p2 += s[i] * q[i];
    s[i] = g[i] * s[i] + k[i] * v;
  }
  return row_sum(p2) + dot * v;
}

// Per-head RMS norm, weight and gate: one wave per (token, head). DELTA: the
// weight is shared by heads and the gate a sigmoid; else a weight per head
// and a silu.
template <typename T, bool DELTA, int PER>
__global__ __launch_bounds__(256) void head_norm_gate_kernel(
    const float* __restrict__ o, const T* __restrict__ norm, const T* __restrict__ gate, T* __restrict__ out,
    int total, RecArgs a, Step step) {
  const int id = blockIdx.x * 4 + (threadIdx.x >> 6), c = (threadIdx.x & 63) * PER;
  if (id >= total) return;
  const int h = id % a.H, tok = id / a.H, s = tok % a.S, b = tok / a.S;
  const bool live = step.slot(b) >= 0 && s < step.len(b, a.S), vec = (a.vdim & 3) == 0;
  const size_t src = ((size_t)tok * a.H + h) * a.vdim;
  float x[PER], g[PER], w[PER], ss = 0.f;
  ld_lane<PER>(o + src, c, live ? a.vdim : 0, vec, x);
  ld_lane<PER>(gate + src, c, a.vdim, vec, g);
  ld_lane<PER>(norm + (DELTA ? 0 : h * a.vdim), c, a.vdim, vec, w);
#pragma unroll
  for (int i = 0; i < PER; ++i) ss += x[i] * x[i];
  const float inv = a.out_scale / sqrtf(wave_sum(ss) / (float)a.vdim + a.eps);
#pragma unroll
  for (int i = 0; i < PER; ++i) x[i] = live ? x[i] * inv * w[i] * (DELTA ? sigmoidf(g[i]) : siluf(g[i])) : 0.f;
  st_lane<PER>(out + (size_t)tok * a.K + a.out_at + h * a.vdim, c, a.vdim, vec && ((a.K | a.out_at) & 3) == 0, x);
}

template <bool DELTA>
static void launch_head_norm_gate(bool bf16, const torch::Tensor& o, const torch::Tensor& norm,
                                  const torch::Tensor& gate, torch::Tensor& out, int heads, const RecArgs& a,
                                  const Step& step, hipStream_t stream) {
#define GATE(T, PER)                                                                                             \
  hipLaunchKernelGGL((head_norm_gate_kernel<T, DELTA, PER>), dim3((heads + 3) / 4), dim3(256), 0, stream,       \
                     (const float*)o.data_ptr(), (const T*)norm.data_ptr(), (const T*)gate.data_ptr(),          \
                     (T*)out.data_ptr(), heads, a, step)
#define GATE_WIDTH(T) \
  if (a.vdim <= 64) GATE(T, 1); else if (a.vdim <= 128) GATE(T, 2); else GATE(T, 4);
  if (bf16) { GATE_WIDTH(bf16_t) } else { GATE_WIDTH(float) }
#undef GATE_WIDTH
#undef GATE
}

// One token of one head, everything from projections to the gated output: a
// block streams the head's state once. DELTA inputs: q/k/v columns of `in0`
// (with their convolutions), beta there too; WKV inputs: r, k, v tensors.
template <typename T, bool DELTA, int RPL>
__global__ __launch_bounds__(256) void rec_decode_kernel(
    const T* __restrict__ in0, const T* __restrict__ in1, const T* __restrict__ in2, const T* __restrict__ w0_,
    const T* __restrict__ w1_, const T* __restrict__ w2_, const T* __restrict__ pre, const T* __restrict__ a_log,
    const T* __restrict__ dt, const T* __restrict__ norm, const T* __restrict__ gate, float* __restrict__ state,
    T* __restrict__ ring, T* __restrict__ out, RecArgs a, Step step) {
  constexpr int DP = 16 * RPL;
  __shared__ __attribute__((aligned(16))) float sq[DP], sk[DP], sg[DP];
  __shared__ float sv[256], so[256], red[16];
  const int h = blockIdx.x, b = blockIdx.y, tid = threadIdx.x, g = h / (a.H / a.G);
  const int slot = step.slot(b);
  T* dst = out + (size_t)b * a.K + a.out_at + h * a.vdim;
  if (slot < 0) {
    if (tid < a.vdim) st(dst + tid, 0.f);
    return;
  }
  const int pos = step.first(b);
  // (dim and vdim are at most 256: one channel a thread)
  float q = 0.f, k = 0.f, dec = 1.f, beta = 0.f, extra = 0.f;
  if (DELTA) {
    const int C = 2 * a.G * a.dim + a.H * a.vdim, qch = g * a.dim + tid, vch = h * a.vdim + tid;
    const T* row = in0 + (size_t)b * a.N;
    T* hist = ring + (size_t)slot * a.taps * C;
    T* now = hist + (size_t)(pos % a.taps) * C;  // a row that no convolution of this step reads
    if (tid < a.dim) {
      q = conv_silu(row, hist, w0_, 0, pos, a.q_at + qch, qch, qch, C, a);
      k = conv_silu(row, hist, w1_, 0, pos, a.k_at + qch, a.G * a.dim + qch, qch, C, a);
      if (h % (a.H / a.G) == 0) {
        now[qch] = row[a.q_at + qch];
        now[a.G * a.dim + qch] = row[a.k_at + qch];
      }
      const int ch = h * a.dim + tid;
      dec = expf(-expf(ld(a_log + h)) * softplusf(ld(pre + (size_t)b * a.H * a.dim + ch) + ld(dt + ch)));
    }
    if (tid < a.vdim) {
      sv[tid] = conv_silu(row, hist, w2_, 0, pos, a.v_at + vch, 2 * a.G * a.dim + vch, vch, C, a);
      now[2 * a.G * a.dim + vch] = row[a.v_at + vch];
    }
    beta = sigmoidf(ld(row + a.b_at + h));
  } else if (tid < a.dim) {
    const size_t src = ((size_t)b * a.H + h) * a.dim + tid;
    q = ld(in0 + src);
    k = ld(in1 + src);
    sv[tid] = ld(in2 + src);
    dec = expf(-expf(ld(pre + src) + ld(w0_ + h * a.dim + tid)));
    extra = q * k * ld(w1_ + h * a.dim + tid);
  }
  float dot;
  if (DELTA) {
    const float qq = wave_sum(q * q), kk = wave_sum(k * k), qk = wave_sum(q * k);
    if ((tid & 63) == 0) { red[tid >> 6] = qq; red[4 + (tid >> 6)] = kk; red[8 + (tid >> 6)] = qk; }
    __syncthreads();
    const float qi = 1.f / sqrtf(red[0] + red[1] + red[2] + red[3] + 1e-6f) / sqrtf((float)a.dim);
    const float ki = 1.f / sqrtf(red[4] + red[5] + red[6] + red[7] + 1e-6f);
    dot = (red[8] + red[9] + red[10] + red[11]) * qi * ki;
    q *= qi;
    k *= ki;
  } else {
    dot = block_sum(extra, red);
  }
  if (tid < DP) { sq[tid] = q; sk[tid] = k; sg[tid] = dec; }
  __syncthreads();
  const int r = tid & 15, cl = tid >> 4;
  float qq[RPL], kk[RPL], gg[RPL];
  load_rows<RPL>(sq, r, qq);
  load_rows<RPL>(sk, r, kk);
  load_rows<RPL>(sg, r, gg);
  float* base = state + ((size_t)slot * a.H + h) * (size_t)a.vdim * DP;
  constexpr int NB = RPL <= 8 ? 4 : 2;  // columns in flight per lane group
  for (int c0 = 0; c0 < a.vdim; c0 += 16 * NB) {
    float s[NB][RPL];
#pragma unroll
    for (int i = 0; i < NB; ++i) {
      const int col = c0 + i * 16 + cl;
      if (col < a.vdim && pos > 0) load_rows<RPL>(base + (size_t)col * DP, r, s[i]);
      else
#pragma unroll
        for (int j = 0; j < RPL; ++j) s[i][j] = 0.f;
    }
#pragma unroll
    for (int i = 0; i < NB; ++i) {
      const int col = c0 + i * 16 + cl;
      const float y = rec_step<DELTA, RPL>(s[i], qq, kk, gg, sv[min(col, a.vdim - 1)], beta, dot);
      if (col < a.vdim) {
        if (r == 0) so[col] = y;
        store_rows<RPL>(base + (size_t)col * DP, r, s[i]);
      }
    }
  }
  __syncthreads();
  const float y = tid < a.vdim ? so[tid] : 0.f;
  const float inv = 1.f / sqrtf(block_sum(y * y, red + 12) / (float)a.vdim + a.eps);
  if (tid < a.vdim) {
    const float gv = ld(gate + ((size_t)b * a.H + h) * a.vdim + tid);
    st(dst + tid, y * inv * ld(norm + (DELTA ? tid : h * a.vdim + tid)) * (DELTA ? sigmoidf(gv) : siluf(gv)) *
                      a.out_scale);
  }
}

// n blends of the current and the previous token: out [n][B,S,D]
template <typename T, int V>
__global__ __launch_bounds__(256) void token_shift_kernel(
    const T* __restrict__ h, const T* __restrict__ mu, T* __restrict__ ring, T* __restrict__ out, int S, int D,
    int M, int n, size_t plane, Step step) {
  const int s = blockIdx.x, b = blockIdx.y;
  const int slot = step.slot(b), len = step.decode ? 1 : step.len(b, S);
  const bool live = slot >= 0 && s < len;
  const int first = live ? step.first(b) : 0;
  const size_t at = ((size_t)b * S + s) * D;
  for (int d = threadIdx.x * V; d < D; d += 256 * V) {
    float x[V], p[V];
#pragma unroll
    for (int i = 0; i < V; ++i) x[i] = p[i] = 0.f;
    if (live) {
      ldv<V>(h + at + d, x);
      if (s > 0) ldv<V>(h + at - D + d, p);
      else if (first > 0) ldv<V>(ring + ((size_t)slot * M + (first - 1) % M) * D + d, p);
      if (step.decode) stv<V>(ring + ((size_t)slot * M + first % M) * D + d, x);  // M >= 2: not the row just read
    }
#pragma unroll
    for (int i = 0; i < V; ++i) p[i] -= x[i];
    for (int j = 0; j < n; ++j) {
      float m[V];
      ldv<V>(mu + (size_t)j * D + d, m);
#pragma unroll
      for (int i = 0; i < V; ++i) m[i] = x[i] + p[i] * m[i];
      stv<V>(out + j * plane + at + d, m);
    }
  }
}

// ===========================================================================
// host side
// ===========================================================================

// what a sublayer's output row is made of: itself, or weighted rows (rows set)
struct Gather { const int* rows; const float* weight; int top, ys; };

template <typename T, int V>
static void launch_norm(const T* y, const Gather& from, float* x, const T* wp, const T* wn, T* h, int copy, int rows,
                        int D, float eps) {
  const int nc = (D + 256 * V - 1) / (256 * V);
#define NORM_CASE(NC)                                                                                              \
  if (nc <= NC) {                                                                                                  \
    hipLaunchKernelGGL((sandwich_norm_kernel<T, V, NC>), dim3(rows), dim3(256), 0, cur_stream(), y, from.rows,     \
                       from.weight, from.top, from.ys, x, wp, wn, h, copy, D, eps);                                \
    return;                                                                                                        \
  }
  NORM_CASE(1) NORM_CASE(2) NORM_CASE(4) NORM_CASE(8) NORM_CASE(16)
#undef NORM_CASE
  TORCH_CHECK(false, "row of ", D, " elements is too long");
}

static OptT norm_host(const OptT& y, Tensor x, const OptT& w_post, const OptT& w_next, double eps, bool copy,
                      const OptT& take, const OptT& weight, torch::ScalarType dt) {
  check_io(x, torch::kFloat32);
  const int D = x.size(-1), rows = x.numel() / D;
  Gather from{nullptr, nullptr, 0, D};
  CHK(!copy || (y && !w_next));
  if (y) {
    check_io(*y, dt);
    CHK(w_post);
    check_io(*w_post, dt);
    CHK(w_post->numel() == D);
  }
  if (take) {
    CHK(y);
    check_io(*take, torch::kInt32);
    if (weight) { check_io(*weight, torch::kFloat32); CHK(weight->numel() == take->numel()); }
    from = Gather{take->data_ptr<int>(), weight ? weight->data_ptr<float>() : nullptr, (int)take->size(-1),
                  (int)y->size(-1)};
    CHK(take->numel() == (int64_t)rows * from.top && from.ys >= D && y->numel() == take->numel() * from.ys);
  } else if (y) {
    CHK(y->numel() == x.numel() && y->size(-1) == D);
  }
  OptT h;
  if (w_next) { check_io(*w_next, dt); CHK(w_next->numel() == D); }
  if (w_next || copy) h = torch::empty(x.sizes(), x.options().dtype(dt));
  if (rows == 0) return h;
  BY_TYPE(dt, {
    const T* yp = y ? P<T>(*y) : nullptr;
    const T* wp = w_post ? P<T>(*w_post) : nullptr;
    const T* wn = w_next ? P<T>(*w_next) : nullptr;
    T* hp = h ? M<T>(*h) : nullptr;
    if (((D | from.ys) & 3) == 0) launch_norm<T, 4>(yp, from, M<float>(x), wp, wn, hp, copy, rows, D, (float)eps);
    else launch_norm<T, 1>(yp, from, M<float>(x), wp, wn, hp, copy, rows, D, (float)eps);
  });
  return h;
}

// take, weight [tokens, top]: y is not yet summed, row take[t, k] counts weight[t, k]
// (no weight: one)
OptT sandwich_norm(Tensor y, Tensor x, Tensor w_post, OptT w_next, double eps, bool copy, OptT take, OptT weight) {
  return norm_host(y, x, w_post, w_next, eps, copy, take, weight, io_type(y));
}

Tensor prenorm(Tensor x, Tensor w, double eps, bool bf16) {
  return *norm_host(c10::nullopt, x, c10::nullopt, w, eps, false, c10::nullopt, c10::nullopt,
                    bf16 ? torch::kBFloat16 : torch::kFloat32);
}

Tensor swiglu_packed(Tensor gu) {
  const auto dt = io_type(gu);
  const int I = gu.size(-1) / 2;
  CHK(gu.size(-1) == 2 * I);
  auto shape = gu.sizes().vec();
  shape.back() = I;
  auto out = torch::empty(shape, gu.options());
  const long long n = out.numel();
  if (n == 0) return out;
  BY_TYPE(dt, {
    if (I % 4 == 0)
      hipLaunchKernelGGL((swiglu_kernel<T, 4>), dim3((n / 4 + 255) / 256), dim3(256), 0, cur_stream(), P<T>(gu), M<T>(out), n, I);
    else
      hipLaunchKernelGGL((swiglu_kernel<T, 1>), dim3((n + 255) / 256), dim3(256), 0, cur_stream(), P<T>(gu), M<T>(out), n, I);
  });
  return out;
}

Tensor tanh_op(Tensor x) {
  const auto dt = io_type(x);
  auto out = torch::empty_like(x);
  const long long n = x.numel();
  if (n == 0) return out;
  BY_TYPE(dt, { hipLaunchKernelGGL((tanh_kernel<T>), dim3((n + 255) / 256), dim3(256), 0, cur_stream(), P<T>(x), M<T>(out), n); });
  return out;
}

static int row_pad(int dim) {
  for (int p : {1, 2, 3, 4, 6, 8, 12, 16})
    if (dim <= 16 * p) return 16 * p;
  TORCH_CHECK(false, "recurrent state with ", dim, " key channels");
}

#define BY_ROWS(dp, ...)                                                                                   \
  switch (dp / 16) {                                                                                       \
    case 1: { constexpr int R = 1; __VA_ARGS__; break; }  case 2: { constexpr int R = 2; __VA_ARGS__; break; }   \
    case 3: { constexpr int R = 3; __VA_ARGS__; break; }  case 4: { constexpr int R = 4; __VA_ARGS__; break; }   \
    case 6: { constexpr int R = 6; __VA_ARGS__; break; }  case 8: { constexpr int R = 8; __VA_ARGS__; break; }   \
    case 12: { constexpr int R = 12; __VA_ARGS__; break; } case 16: { constexpr int R = 16; __VA_ARGS__; break; } \
    default: TORCH_CHECK(false, "padded key channels ", dp);                                               \
  }

static int64_t chunk_count(int S) { return (S + CHUNK - 1) / CHUNK; }
static int64_t chunk_size(bool delta, int dp) { return delta ? 49 * dp + 512 : 33 * dp + 256; }

template <bool DELTA>
static void launch_scan(int B, const Tensor& factors, const Tensor& v, Tensor& state, Tensor& o, const RecArgs& a,
                        const Step& step) {
  const int groups = (a.vdim + 15) / 16 * a.H * B;  // of 16 columns
#define SCAN(KS)                                                                                                    \
  hipLaunchKernelGGL((chunk_scan_kernel<DELTA, R, KS>), dim3((a.vdim + 64 / KS - 1) / (64 / KS), a.H, B), dim3(256), 0, \
                     cur_stream(), P<float>(factors), P<float>(v), M<float>(state), M<float>(o),                    \
                     (int)chunk_count(a.S), a, step)
  BY_ROWS(a.dp, {
    constexpr int TWO = R % 2 ? 1 : 2, FOUR = R % 4 ? TWO : 4;
    // split channels while the chip's 1024 SIMDs are not covered
    if (groups * 4 <= 1024) SCAN(FOUR);
    else if (groups * 2 <= 1024) SCAN(TWO);
    else SCAN(1);
  });
#undef SCAN
}

// channels per lane and, for the delta rule, taps as template arguments
template <typename T, bool DELTA, int TAPS>
static void launch_prep_width(int B, const T* x0, const T* x1, const T* x2, const T* c0, const T* c1, const T* c2,
                              const T* pre, const T* d0, const T* d1, const T* ring, Tensor& factors, Tensor& v,
                              const RecArgs& a, const Step& step) {
  const int chunks = chunk_count(a.S), widest = std::max(a.vdim, a.dp);
  TORCH_CHECK(chunks <= 65535 && B <= 65535, "a prefill step of ", B, " x ", a.S, " tokens is too large");
  const dim3 grid(a.H, chunks, B);
  const size_t lds = (3 * CHUNK * (a.dp + 4) + 512 + CHUNK) * sizeof(float);
#define PREP(PER)                                                                                              \
  hipLaunchKernelGGL((chunk_prep_kernel<T, DELTA, TAPS, PER>), grid, dim3(256), lds, cur_stream(), x0, x1, x2, c0, c1, \
                     c2, pre, d0, d1, ring, M<float>(factors), M<float>(v), chunks, a, step)
  if (widest <= 64) PREP(1);
  else if (widest <= 128) PREP(2);
  else PREP(4);
#undef PREP
}

template <typename T>
static void remember(const Tensor& src, Tensor& ring, int B, int S, int N, Columns cols, const Step& step) {
  const int Mr = ring.size(1), C = ring.size(2);
  hipLaunchKernelGGL((remember_kernel<T>), dim3(std::min(Mr, S), B), dim3(256), 0, cur_stream(), P<T>(src), M<T>(ring), S, N, Mr, C, cols, step);
}

void delta_rule(Tensor proj, int64_t q_at, int64_t k_at, int64_t v_at, int64_t b_at, int64_t H, int64_t G, int64_t dim,
                int64_t vdim, Tensor qc, Tensor kcv, Tensor vcv, Tensor pre, Tensor pre_gate, Tensor a_log, Tensor dt_,
                Tensor norm, double eps, Tensor state, Tensor ring, OptT slots, OptT positions, OptT lens,
                int64_t start, bool decode, Tensor out, int64_t out_at, double out_scale) {
  const auto dt = io_type(proj);
  CHK(proj.dim() == 3 && out.dim() == 3 && out.size(0) == proj.size(0) && out.size(1) == proj.size(1));
  for (const Tensor& t : {qc, kcv, vcv, pre, pre_gate, a_log, dt_, norm, ring, out}) check_io(t, dt);
  check_io(state, torch::kFloat32);
  const int B = proj.size(0), S = proj.size(1), N = proj.size(2), taps = qc.size(-1);
  const int dp = row_pad(dim), C = 2 * G * dim + H * vdim;
  CHK(H > 0 && G > 0 && H % G == 0 && dim > 0 && vdim > 0 && vdim <= 256 && taps > 0);
  CHK(q_at + G * dim <= N && k_at + G * dim <= N && v_at + H * vdim <= N && b_at + H <= N);
  CHK(out_at + H * vdim <= out.size(2) && (!decode || S == 1));
  CHK(qc.numel() == G * dim * taps && kcv.numel() == G * dim * taps && vcv.numel() == H * vdim * taps);
  CHK(pre.numel() == (int64_t)B * S * H * dim && pre_gate.numel() == (int64_t)B * S * H * vdim);
  CHK(a_log.numel() == H && dt_.numel() == H * dim && norm.numel() == vdim);
  CHK(state.dim() == 4 && state.size(1) == H && state.size(2) == vdim && state.size(3) == dp);
  CHK(ring.dim() == 3 && ring.size(0) == state.size(0) && ring.size(1) == taps && ring.size(2) == C);
  CHK(slots || B <= state.size(0));
  if (B == 0 || S == 0) return;
  const Step step = make_step(slots, positions, lens, start, decode, B);
  RecArgs a{S, (int)H, (int)G, N, (int)out.size(2), (int)dim, (int)vdim, dp, taps, (int)q_at, (int)k_at, (int)v_at,
            (int)b_at, (int)out_at, (float)eps, (float)out_scale};
  const hipStream_t stream = cur_stream();
  if (decode) {
    BY_TYPE(dt, BY_ROWS(dp, {
      hipLaunchKernelGGL((rec_decode_kernel<T, true, R>), dim3(H, B), dim3(256), 0, stream, P<T>(proj), nullptr,
                         nullptr, P<T>(qc), P<T>(kcv), P<T>(vcv), P<T>(pre), P<T>(a_log), P<T>(dt_), P<T>(norm),
                         P<T>(pre_gate), M<float>(state), M<T>(ring), M<T>(out), a, step);
    }));
    return;
  }
  auto factors = f32(proj, {B, chunk_count(S), H, chunk_size(true, dp)});
  auto v = f32(proj, {B, S, H, vdim}), o = f32(proj, {B, S, H, vdim});
  const int heads = B * S * (int)H;
  BY_TYPE(dt, {
    auto prep = [&](auto launch) {
      launch(B, P<T>(proj), (const T*)nullptr, (const T*)nullptr, P<T>(qc), P<T>(kcv), P<T>(vcv), P<T>(pre),
             P<T>(a_log), P<T>(dt_), (const T*)P<T>(ring), factors, v, a, step);
    };
    if (taps == 2) prep(launch_prep_width<T, true, 2>);
    else if (taps == 3) prep(launch_prep_width<T, true, 3>);
    else if (taps == 4) prep(launch_prep_width<T, true, 4>);
    else prep(launch_prep_width<T, true, 0>);
    remember<T>(proj, ring, B, S, N, Columns{{(int)q_at, (int)k_at, (int)v_at}, {(int)(G * dim), (int)(G * dim), (int)(H * vdim)}}, step);
  });
  launch_scan<true>(B, factors, v, state, o, a, step);
  launch_head_norm_gate<true>(dt == torch::kBFloat16, o, norm, pre_gate, out, heads, a, step, stream);
}

Tensor wkv(Tensor r, Tensor k_, Tensor v_, Tensor gate, Tensor pre, Tensor w0, Tensor u, Tensor norm, int64_t H,
           int64_t dim, double eps, Tensor state, OptT slots, OptT positions, OptT lens, int64_t start, bool decode) {
  const auto dt = io_type(r);
  const int dp = row_pad(dim);
  CHK(r.dim() == 3 && r.size(2) == H * dim && H > 0 && dim > 0);
  for (const Tensor& t : {k_, v_, gate, pre}) { check_io(t, dt); CHK(t.sizes() == r.sizes()); }
  for (const Tensor& t : {w0, u, norm}) { check_io(t, dt); CHK(t.numel() == H * dim); }
  check_io(state, torch::kFloat32);
  const int B = r.size(0), S = r.size(1);
  CHK(state.dim() == 4 && state.size(1) == H && state.size(2) == dim && state.size(3) == dp);
  CHK((slots || B <= state.size(0)) && (!decode || S == 1));
  auto out = torch::empty_like(r);
  if (B == 0 || S == 0) return out;
  const Step step = make_step(slots, positions, lens, start, decode, B);
  RecArgs a{S, (int)H, (int)H, 0, (int)(H * dim), (int)dim, (int)dim, dp, 1, 0, 0, 0, 0, 0, (float)eps, 1.f};
  const hipStream_t stream = cur_stream();
  if (decode) {
    BY_TYPE(dt, BY_ROWS(dp, {
      hipLaunchKernelGGL((rec_decode_kernel<T, false, R>), dim3(H, B), dim3(256), 0, stream, P<T>(r), P<T>(k_),
                         P<T>(v_), P<T>(w0), P<T>(u), nullptr, P<T>(pre), nullptr, nullptr, P<T>(norm), P<T>(gate),
                         M<float>(state), nullptr, M<T>(out), a, step);
    }));
    return out;
  }
  auto factors = f32(r, {B, chunk_count(S), H, chunk_size(false, dp)});
  auto v = f32(r, {B, S, H, dim}), o = f32(r, {B, S, H, dim});
  const int heads = B * S * (int)H;
  BY_TYPE(dt, {
    const T* none = nullptr;
    launch_prep_width<T, false, 1>(B, P<T>(r), P<T>(k_), P<T>(v_), none, none, none, P<T>(pre), P<T>(w0), P<T>(u), none,
                                   factors, v, a, step);
  });
  launch_scan<false>(B, factors, v, state, o, a, step);
  launch_head_norm_gate<false>(dt == torch::kBFloat16, o, norm, gate, out, heads, a, step, stream);
  return out;
}

Tensor token_shift(Tensor h, Tensor mu, Tensor ring, OptT slots, OptT positions, OptT lens, int64_t start, bool decode) {
  const auto dt = io_type(h);
  check_io(mu, dt);
  check_io(ring, dt);
  CHK(h.dim() == 3 && mu.dim() == 2 && mu.size(1) == h.size(2));
  const int B = h.size(0), S = h.size(1), D = h.size(2), n = mu.size(0);
  CHK(ring.dim() == 3 && ring.size(1) >= 2 && ring.size(2) == D && (slots || B <= ring.size(0)) && (!decode || S == 1));
  auto out = torch::empty({n, B, S, D}, h.options());
  if (B == 0 || S == 0) return out;
  const Step step = make_step(slots, positions, lens, start, decode, B);
  BY_TYPE(dt, {
    if (D % 4 == 0)
      hipLaunchKernelGGL((token_shift_kernel<T, 4>), dim3(S, B), dim3(256), 0, cur_stream(), P<T>(h), P<T>(mu),
                         M<T>(ring), M<T>(out), S, D, (int)ring.size(1), n, (size_t)B * S * D, step);
    else
      hipLaunchKernelGGL((token_shift_kernel<T, 1>), dim3(S, B), dim3(256), 0, cur_stream(), P<T>(h), P<T>(mu),
                         M<T>(ring), M<T>(out), S, D, (int)ring.size(1), n, (size_t)B * S * D, step);
    if (!decode) remember<T>(h, ring, B, S, D, Columns{{0, 0, 0}, {D, 0, 0}}, step);
  });
  return out;
}

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.def("prenorm", &prenorm, "RMS norm with a (1+w) weight of the fp32 stream");
  m.def("sandwich_norm", &sandwich_norm, "stream += norm(y); norm or copy of the stream for the next sublayer",
        py::arg("y"), py::arg("x"), py::arg("w_post"), py::arg("w_next"), py::arg("eps"), py::arg("copy") = false,
        py::arg("take") = py::none(), py::arg("weight") = py::none());
  m.def("swiglu_packed", &swiglu_packed, "SwiGLU on a packed projection, any width, bf16 or fp32");
  m.def("tanh", &tanh_op, "tanh with fp32 math");
  m.def("delta_rule", &delta_rule, "gated delta rule with short convolutions and per-channel decay");
  m.def("wkv", &wkv, "decayed outer-product memory with a current-token bonus");
  m.def("token_shift", &token_shift, "blends of the current and the previous token");
}

