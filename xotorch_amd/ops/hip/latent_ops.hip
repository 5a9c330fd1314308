// CDNA4 (gfx950) kernels of latent attention of any size: keys and values of
// all heads come out of one latent of R channels per token, plus r rotated key
// channels that the heads share; only these are cached.
//   - latent_append: RMS norm of the latent, rotation (neighbouring pairs) of
//     the shared key part and of every query, cache append
//   - prompts: latents of all earlier tokens are expanded by a GEMM;
//     pack_heads lays its output out for causal_attn (attn_rows.hip)
//   - decode: the expansion folds into query and output, so one pass over the
//     latents serves all heads (latent_decode); gather_heads lays the expanded
//     output out by token, times its gates
// A head may have a sink, a learned score that joins the softmax's denominator.
//
// Cache, bf16: keys [slots][rows/16][KC][64][8] over R + r channels and values
// [slots][VG][rows/32][64][8] over R channels, both in the fragment order of
// common.h (one head). fp32: plain rows.

#include "common.h"

struct LatArgs {
  int S, H, N, q_at, c_at;   // tokens, heads, projection width and columns
  int d, r, R;               // unrotated and rotated dims of a head, latent
  int qd;                    // dims of a query row (prompts, padded)
  float eps;
};

DEVINL void rotate(float u, float v, float angle, float* o) {
  float s, c;
  sincosf(angle, &s, &c);
  o[0] = u * c - v * s;
  o[1] = v * c + u * s;
}

// One block per token. Prompts: queries [B,S,H,qd] as [d | r rotated | 0],
// latents and shared keys also into workspace rows [B,rows,R] and [B,rows,r]
// at hist + s. Decode: queries split into qn [H,B,d] and qr [B,H,r].
template <typename T>
__global__ __launch_bounds__(256) void latent_append_kernel(
    const T* __restrict__ proj, const T* __restrict__ norm, const float* __restrict__ freq, T* __restrict__ qw,
    T* __restrict__ qn, T* __restrict__ qr, T* __restrict__ kc, T* __restrict__ vc, T* __restrict__ lw,
    T* __restrict__ rw, KVShape cache, int ws_rows, int hist, LatArgs a, Step step) {
  const int s = blockIdx.x, b = blockIdx.y, B = gridDim.y;
  const int slot = step.slot(b), len = step.decode ? 1 : step.len(b, a.S);
  typedef Layout<T> L;
  const bool live = s < len && slot >= 0;
  const size_t tok = (size_t)b * a.S + s;
  const T* row = proj + tok * a.N;
  const int pos = live ? step.first(b) + s : 0, half = a.r >> 1;
  const bool keep = live && pos < cache.rows;
  __shared__ float red[4];
  // queries
  for (int i = threadIdx.x; i < a.H * a.d; i += 256) {
    const int h = i / a.d, d = i - h * a.d;
    const float f = live ? ld(row + a.q_at + h * (a.d + a.r) + d) : 0.f;
    if (qw) st(qw + (tok * a.H + h) * a.qd + d, f);
    else st(qn + ((size_t)h * B + b) * a.d + d, f);
  }
  for (int i = threadIdx.x; i < a.H * half; i += 256) {
    const int h = i / half, j = i - h * half;
    float o[2] = {0.f, 0.f};
    if (live) {
      const T* q = row + a.q_at + h * (a.d + a.r) + a.d + 2 * j;
      rotate(ld(q), ld(q + 1), (float)pos * freq[j], o);
    }
    T* dst = qw ? qw + (tok * a.H + h) * a.qd + a.d + 2 * j : qr + ((size_t)b * a.H + h) * a.r + 2 * j;
    st(dst, o[0]);
    st(dst + 1, o[1]);
  }
  const int pad = qw ? a.qd - a.d - a.r : 0;
  for (int i = threadIdx.x; i < a.H * pad; i += 256) {
    const int h = i / pad;
    st(qw + (tok * a.H + h) * a.qd + a.d + a.r + i - h * pad, 0.f);
  }
  // latent
  float ss = 0.f;
  for (int i = threadIdx.x; i < a.R; i += 256) {
    const float f = live ? ld(row + a.c_at + i) : 0.f;
    ss += f * f;
  }
  const float inv = 1.f / sqrtf(block_sum(ss, red) / (float)a.R + a.eps);
  const int kdims = sizeof(T) == 2 ? cache.kc * 32 : cache.dim, vdims = sizeof(T) == 2 ? cache.vg * 16 : cache.vdim;
  T* kb = kc + L::kbase(cache, max(slot, 0));
  T* vb = vc + L::vbase(cache, max(slot, 0));
  for (int i = threadIdx.x; i < max(vdims, a.R); i += 256) {
    const float f = live && i < a.R ? ld(row + a.c_at + i) * inv * ld(norm + i) : 0.f;
    if (keep) {
      if (i < a.R) st(kb + L::k(cache, pos, i), f);
      st(vb + L::v(cache, pos, i), f);
    }
    if (lw && i < a.R) st(lw + ((size_t)b * ws_rows + hist + s) * a.R + i, f);
  }
  for (int j = threadIdx.x; j < half; j += 256) {
    float o[2] = {0.f, 0.f};
    if (live) {
      const T* k = row + a.c_at + a.R + 2 * j;
      rotate(ld(k), ld(k + 1), (float)pos * freq[j], o);
    }
#pragma unroll
    for (int e = 0; e < 2; ++e) {
      if (keep) st(kb + L::k(cache, pos, a.R + 2 * j + e), o[e]);
      if (rw) st(rw + ((size_t)b * ws_rows + hist + s) * a.r + 2 * j + e, o[e]);
    }
  }
  for (int i = a.R + a.r + threadIdx.x; i < kdims; i += 256)
    if (keep) st(kb + L::k(cache, pos, i), 0.f);
}

// Cached latents and shared keys of positions [0, hist) -> workspace rows.
template <typename T>
__global__ __launch_bounds__(256) void latent_history_kernel(
    const T* __restrict__ kc, T* __restrict__ lw, T* __restrict__ rw, KVShape cache, int ws_rows, int R, int r,
    Step step) {
  const int row = blockIdx.x, b = blockIdx.y, slot = step.slot(b);
  const T* kb = kc + Layout<T>::kbase(cache, max(slot, 0));
  for (int i = threadIdx.x; i < R + r; i += 256) {
    const T f = slot < 0 ? (T)0 : kb[Layout<T>::k(cache, row, i)];
    if (i < R) lw[((size_t)b * ws_rows + row) * R + i] = f;
    else rw[((size_t)b * ws_rows + row) * r + i - R] = f;
  }
}

// Expanded rows kv [B,rows,H*d + H*e] and shared keys [B,rows,r] -> keys and
// values of every head in the order of common.h. A block packs 32 rows of one
// head; rows past `rows` are zero.
template <typename T>
__global__ __launch_bounds__(256) void pack_heads_kernel(
    const T* __restrict__ kv, const T* __restrict__ rot, T* __restrict__ kw, T* __restrict__ vw, KVShape ws, int rows,
    int H, int d, int r, int e) {
  typedef Layout<T> L;
  const int r0 = blockIdx.x * 32, h = blockIdx.y, b = blockIdx.z;
  const size_t N = (size_t)H * (d + e);
  T* kb = kw + L::kbase(ws, (size_t)b * H + h);
  T* vb = vw + L::vbase(ws, (size_t)b * H + h);
  const int kdims = sizeof(T) == 2 ? ws.kc * 32 : ws.dim, vdims = sizeof(T) == 2 ? ws.vg * 16 : ws.vdim;
  const bool vec = sizeof(T) == 2 && ((d | r) & 7) == 0;
  if (vec) {  // 8 channels of a row lie together on both sides
    typedef __attribute__((ext_vector_type(4))) float piece;
    const int pieces = kdims >> 3;
    for (int i = threadIdx.x; i < 32 * pieces; i += 256) {
      const int row = r0 + i / pieces, c = i % pieces * 8;
      piece v = (piece)(0.f);
      if (row < rows) {
        if (c < d) v = *(const piece*)(kv + ((size_t)b * rows + row) * N + (size_t)h * d + c);
        else if (c < d + r) v = *(const piece*)(rot + ((size_t)b * rows + row) * r + c - d);
      }
      *(piece*)(kb + L::k(ws, row, c)) = v;
    }
  } else {
    for (int i = threadIdx.x; i < 32 * kdims; i += 256) {
      const int row = r0 + i / kdims, c = i % kdims;
      if (row >= ws.rows) continue;
      T v = (T)0;
      if (row < rows) {
        if (c < d) v = kv[((size_t)b * rows + row) * N + (size_t)h * d + c];
        else if (c < d + r) v = rot[((size_t)b * rows + row) * r + c - d];
      }
      kb[L::k(ws, row, c)] = v;
    }
  }
  // four rows of a column lie together in the packed values
  for (int i = threadIdx.x; i < 8 * vdims; i += 256) {
    const int row = r0 + i / vdims * 4, c = i % vdims;
    T v[4];
#pragma unroll
    for (int j = 0; j < 4; ++j)
      v[j] = row + j < rows && c < e ? kv[((size_t)b * rows + row + j) * N + (size_t)H * d + (size_t)h * e + c] : (T)0;
    if (sizeof(T) == 2) {
      ushort4_t p;
#pragma unroll
      for (int j = 0; j < 4; ++j) p[j] = (unsigned short)v[j];
      *(ushort4_t*)(vb + L::v(ws, row, c)) = p;
    } else {
#pragma unroll
      for (int j = 0; j < 4; ++j)
        if (row + j < ws.rows) vb[L::v(ws, row + j, c)] = v[j];
    }
  }
}

// Decode: a block takes up to 16 heads of one row and a part of its tokens,
// 128 at a time: each wave scores 32 of them, then owns a quarter of the output
// channels over all 128. GW: 16-channel groups a wave owns at most.
template <int GW>
__global__ __launch_bounds__(256) void latent_decode_kernel(
    const bf16_t* __restrict__ ql, const bf16_t* __restrict__ qr, const bf16_t* __restrict__ kc_,
    const bf16_t* __restrict__ vc_, const bf16_t* __restrict__ sinks, bf16_t* __restrict__ out,
    float* __restrict__ part, int splits, KVShape cache, float scale, int H, int R, int r, Step step) {
  extern __shared__ __attribute__((aligned(16))) bf16_t q[];  // [16][kc*32 + 8]
  __shared__ __attribute__((aligned(16))) bf16_t probs[16][128 + 8];
  __shared__ float tops[4][16], sums[4][16];
  const int split = blockIdx.x, h0 = blockIdx.y * 16, b = blockIdx.z, B = gridDim.z;
  const int nh = min(16, H - h0), slot = step.slot(b);
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, col = lane & 15, quad = lane >> 4;
  if (slot < 0) {
    if (!part)
      for (int i = threadIdx.x; i < nh * R; i += 256) st(out + ((size_t)(h0 + i / R) * B + b) * R + i % R, 0.f);
    return;
  }
  const int dims = cache.kc * 32, qs = dims + 8;
  {  // 16 threads a head
    const int hh = threadIdx.x >> 4, h = h0 + min(hh, nh - 1);
    const bf16_t *l = ql + ((size_t)h * B + b) * R, *t = qr + ((size_t)b * H + h) * r;
    if (((R | r) & 7) == 0) {
      for (int c = (threadIdx.x & 15) * 8; c < dims; c += 128) {
        floatx4 v = (floatx4)(0.f);
        if (c < R) v = *(const floatx4*)(l + c);
        else if (c < R + r) v = *(const floatx4*)(t + c - R);
        *(floatx4*)(q + hh * qs + c) = v;
      }
    } else {
      for (int c = threadIdx.x & 15; c < dims; c += 16) q[hh * qs + c] = c < R ? l[c] : c < R + r ? t[c - R] : (bf16_t)0;
    }
  }
  __syncthreads();
  const int seen = min(step.first(b) + 1, cache.rows), ntiles = (seen + 31) >> 5;
  const int per = ((ntiles + splits - 1) / splits + 3) & ~3;  // whole groups of four tiles
  const int begin = split * per, end = min(ntiles, begin + per);
  const int gw = (cache.vg + 3) >> 2, g0 = wave * gw, ng = max(0, min(gw, cache.vg - g0));
  const bf16_t* kb = kc_ + Layout<bf16_t>::kbase(cache, slot);
  const bf16_t* vb = vc_ + Layout<bf16_t>::vbase(cache, slot);
  const size_t vstride = (size_t)(cache.rows >> 5) * 512;
  float m = -1e30f, l = 0.f;
  floatx4 o[GW];
#pragma unroll
  for (int i = 0; i < GW; ++i) o[i] = (floatx4)(0.f);
  for (int t4 = begin; t4 < end; t4 += 4) {
    const int tile = t4 + wave;
    // values of two tiles are on their way before the scores are needed; groups
    // past the wave's own are read again and dropped
    bf16x8 vf[2][GW];
    auto load_values = [&](int w) {
      const bf16_t* v0 = vb + (size_t)min(t4 + w, end - 1) * 512 + lane * 8;
#pragma unroll
      for (int i = 0; i < GW; ++i) vf[w & 1][i] = *(const bf16x8*)(v0 + min(g0 + i, cache.vg - 1) * vstride);
    };
    floatx4 sc[2] = {(floatx4)(0.f), (floatx4)(0.f)};
    if (tile < end) {
      const bf16_t* k0 = kb + (size_t)tile * 2 * cache.kc * 512 + lane * 8;
      const bf16_t* k1 = k0 + (size_t)cache.kc * 512;
      auto run = [&](int c, auto count) {  // `count` pieces of 32 channels, loads first
        constexpr int N = decltype(count)::value;
        bf16x8 f0[N], f1[N];
#pragma unroll
        for (int u = 0; u < N; ++u) {
          f0[u] = *(const bf16x8*)(k0 + (c + u) * 512);
          f1[u] = *(const bf16x8*)(k1 + (c + u) * 512);
        }
#pragma unroll
        for (int u = 0; u < N; ++u) {
          const bf16x8 qf = *(const bf16x8*)(q + col * qs + (c + u) * 32 + quad * 8);
          sc[0] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(f0[u], qf, sc[0], 0, 0, 0);
          sc[1] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(f1[u], qf, sc[1], 0, 0, 0);
        }
      };
      int c = 0;
      for (; c + 9 <= cache.kc; c += 9) run(c, std::integral_constant<int, 9>());
      for (; c < cache.kc; ++c) run(c, std::integral_constant<int, 1>());
    }
    load_values(0);
    load_values(1);
    float top = -1e30f;
#pragma unroll
    for (int hf = 0; hf < 2; ++hf)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const bool on = tile < end && tile * 32 + hf * 16 + quad * 4 + i < seen;
        sc[hf][i] = on ? sc[hf][i] * scale : -INFINITY;
        top = fmaxf(top, sc[hf][i]);
      }
    top = fmaxf(top, __shfl_xor(top, 16));
    top = fmaxf(top, __shfl_xor(top, 32));
    if (quad == 0) tops[wave][col] = top;
    __syncthreads();
    top = fmaxf(fmaxf(fmaxf(tops[0][col], tops[1][col]), fmaxf(tops[2][col], tops[3][col])), m);
    const float al = __expf(m - top);
    m = top;
    l *= al;
    // probabilities in the order of the packed values: lane's 8 are together
    ushort4_t pk[2];
#pragma unroll
    for (int hf = 0; hf < 2; ++hf)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const float p = __expf(sc[hf][i] - top);
        l += p;
        pk[hf][i] = f2b(p);
      }
    *(ushort4_t*)&probs[col][wave * 32 + quad * 8] = pk[0];
    *(ushort4_t*)&probs[col][wave * 32 + quad * 8 + 4] = pk[1];
    __syncthreads();
#pragma unroll
    for (int i = 0; i < GW; ++i) o[i] *= al;
    // all four: tiles past the end weigh nothing, and without branches between
    // them the products follow each other
#pragma unroll
    for (int w = 0; w < 4; ++w) {
      const bf16x8 pf = *(const bf16x8*)&probs[col][w * 32 + quad * 8];
#pragma unroll
      for (int i = 0; i < GW; ++i) o[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf[w & 1][i], pf, o[i], 0, 0, 0);
      if (w < 2) load_values(w + 2);
    }
    // the next round's writes to `tops` are two barriers behind these reads;
    // those to `probs` are one behind
  }
  l += __shfl_xor(l, 16);
  l += __shfl_xor(l, 32);
  if (quad == 0) sums[wave][col] = l;
  __syncthreads();
  const float sum = sums[0][col] + sums[1][col] + sums[2][col] + sums[3][col];
  if (col >= nh) return;
  const int h = h0 + col;
  if (part) {
    float* p = part + (((size_t)b * splits + split) * H + h) * (R + 2);
    if (wave == 0 && quad == 0) { p[0] = m; p[1] = sum; }
#pragma unroll
    for (int i = 0; i < GW; ++i)
      if (i < ng)
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          const int c = (g0 + i) * 16 + quad * 4 + j;
          if (c < R) p[2 + c] = o[i][j];
        }
  } else {
    const float f = 1.f / (sum + (sinks ? __expf(ld(sinks + h) - m) : 0.f));
#pragma unroll
    for (int i = 0; i < GW; ++i)
      if (i < ng)
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          const int c = (g0 + i) * 16 + quad * 4 + j;
          if (c < R) st(out + ((size_t)h * B + b) * R + c, o[i][j] * f);
        }
  }
}

__global__ __launch_bounds__(256) void latent_merge_kernel(const float* __restrict__ part,
                                                           const bf16_t* __restrict__ sinks, bf16_t* __restrict__ out,
                                                           int splits, int H, int R, Step step) {
  extern __shared__ float fac[];  // [splits]
  const int h = blockIdx.x, b = blockIdx.y, B = gridDim.y;
  const bool live = step.slot(b) >= 0;
  const float* p0 = part + ((size_t)b * splits * H + h) * (R + 2);
  const size_t stride = (size_t)H * (R + 2);
  if (live && threadIdx.x < 64) {
    float M = -1e30f, L = 0.f;
    for (int s = threadIdx.x; s < splits; s += 64) M = fmaxf(M, p0[s * stride]);
#pragma unroll
    for (int x = 32; x > 0; x >>= 1) M = fmaxf(M, __shfl_xor(M, x));
    for (int s = threadIdx.x; s < splits; s += 64) {
      fac[s] = __expf(p0[s * stride] - M);
      L += fac[s] * p0[s * stride + 1];
    }
    L = 1.f / (wave_sum(L) + (sinks ? __expf(ld(sinks + h) - M) : 0.f));
    for (int s = threadIdx.x; s < splits; s += 64) fac[s] *= L;
  }
  __syncthreads();
  for (int c = threadIdx.x; c < R; c += 256) {
    float O = 0.f;
    if (live)
#pragma unroll 8
      for (int s = 0; s < splits; ++s) O += fac[s] * p0[s * stride + 2 + c];
    st(out + ((size_t)h * B + b) * R + c, O);
  }
}

// 32-bit decode: one block per (row, head), plain two-pass softmax over rows
// of the cache through a running maximum; lanes over tokens, then over channels.
__global__ __launch_bounds__(256) void latent_decode_f32_kernel(
    const float* __restrict__ ql, const float* __restrict__ qr, const float* __restrict__ kc,
    const float* __restrict__ vc, const float* __restrict__ sinks, float* __restrict__ out, KVShape cache, float scale,
    int H, int R, int r, Step step) {
  extern __shared__ float lds[];  // query [R + r], output [R]
  __shared__ float prob[256], red[8];
  const int h = blockIdx.x, b = blockIdx.y, B = gridDim.y, slot = step.slot(b), tid = threadIdx.x;
  float* dst = out + ((size_t)h * B + b) * R;
  if (slot < 0) {
    for (int c = tid; c < R; c += 256) dst[c] = 0.f;
    return;
  }
  float *q = lds, *acc = lds + R + r;
  for (int c = tid; c < R + r; c += 256) q[c] = c < R ? ql[((size_t)h * B + b) * R + c] : qr[((size_t)b * H + h) * r + c - R];
  for (int c = tid; c < R; c += 256) acc[c] = 0.f;
  __syncthreads();
  const float* kb = kc + Layout<float>::kbase(cache, slot);
  const float* vb = vc + Layout<float>::vbase(cache, slot);
  const int seen = min(step.first(b) + 1, cache.rows);
  float m = -1e30f, l = 0.f;
  for (int p0 = 0; p0 < seen; p0 += 256) {
    float sc = -INFINITY;
    if (p0 + tid < seen) {
      const float* row = kb + (size_t)(p0 + tid) * cache.dim;
      float dot = 0.f;
      for (int c = 0; c < R + r; ++c) dot += q[c] * row[c];
      sc = dot * scale;
    }
    float top = sc;
#pragma unroll
    for (int x = 32; x > 0; x >>= 1) top = fmaxf(top, __shfl_xor(top, x));
    if ((tid & 63) == 0) red[tid >> 6] = top;
    __syncthreads();
    top = fmaxf(fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3])), m);
    const float al = expf(m - top), e = expf(sc - top);
    m = top;
    prob[tid] = e;
    l = l * al + block_sum(e, red + 4);  // its barrier also publishes prob
    const int n = min(256, seen - p0);
    for (int c = tid; c < R; c += 256) {
      float f = acc[c] * al;
      for (int j = 0; j < n; ++j) f += prob[j] * vb[(size_t)(p0 + j) * cache.vdim + c];
      acc[c] = f;
    }
    __syncthreads();
  }
  if (sinks) l += expf(sinks[h] - m);
  for (int c = tid; c < R; c += 256) dst[c] = acc[c] / l;
}

// o [H,B,e] -> columns out_at.. of out [B,1,K], times the sigmoid of the
// columns g_at.. of gates [B,1,N]
template <typename T, int V>
__global__ __launch_bounds__(256) void gather_heads_kernel(const T* __restrict__ o, const T* __restrict__ gates,
                                                           T* __restrict__ out, int B, int HE, int e, int N, int g_at,
                                                           int K, int out_at, float scale) {
  const int c = (blockIdx.x * 256 + threadIdx.x) * V, b = blockIdx.y;
  if (c >= HE) return;
  float v[V], g[V];
  ldv<V>(o + ((size_t)(c / e) * B + b) * e + c % e, v);
  if (gates) ldv<V>(gates + (size_t)b * N + g_at + c, g);
#pragma unroll
  for (int i = 0; i < V; ++i) v[i] *= gates ? scale * sigmoidf(g[i]) : scale;
  stv<V>(out + (size_t)b * K + out_at + c, v);
}

// ===========================================================================
// host side
// ===========================================================================

static KVShape cache_shape(bool bf, int R, int r, const Tensor& kc, const Tensor& vc) {
  KVShape c{R + r, R, (R + r + 31) / 32, (R + 15) / 16, 0, INT_MAX};
  CHK(kc.size(0) == vc.size(0));
  if (bf) {
    CHK(kc.dim() == 5 && vc.dim() == 5 && kc.size(2) == c.kc && vc.size(1) == c.vg);
    c.rows = kc.size(1) * 16;
    CHK(c.rows % 32 == 0 && vc.size(2) * 32 == c.rows);
  } else {
    CHK(kc.dim() == 3 && vc.dim() == 3 && kc.size(2) == R + r && vc.size(2) == R && kc.size(1) == vc.size(1));
    c.rows = kc.size(1);
  }
  CHK(c.rows > 0);
  return c;
}

static LatArgs lat_args(const Tensor& proj, int64_t q_at, int64_t c_at, int64_t H, int64_t d, int64_t r, int64_t R,
                        const Tensor& norm, const Tensor& freq, int qd, double eps) {
  const auto dt = io_type(proj);
  check_io(norm, dt);
  check_io(freq, torch::kFloat32);
  CHK(proj.dim() == 3 && H > 0 && d > 0 && R > 0 && r >= 0 && r % 2 == 0 && norm.numel() == R && freq.numel() == r / 2);
  CHK(q_at + H * (d + r) <= proj.size(2) && c_at + R + r <= proj.size(2) && proj.size(0) <= 65535);
  return LatArgs{(int)proj.size(1), (int)H, (int)proj.size(2), (int)q_at, (int)c_at, (int)d, (int)r, (int)R, qd, (float)eps};
}

// Prompts: -> queries [B,S,H,qd], latents [B,rows,R], shared keys [B,rows,r]
// of positions [0, start + S).
std::vector<Tensor> latent_append(Tensor proj, int64_t q_at, int64_t c_at, int64_t H, int64_t d, int64_t r, int64_t R,
                                  Tensor norm, Tensor freq, double eps, Tensor kc, Tensor vc, OptT slots, OptT lens,
                                  int64_t start) {
  const auto dt = io_type(proj);
  const bool bf = dt == torch::kBFloat16;
  check_io(kc, dt);
  check_io(vc, dt);
  const int qd = bf ? ((int)(d + r) + 31) / 32 * 32 : (int)(d + r);
  const LatArgs a = lat_args(proj, q_at, c_at, H, d, r, R, norm, freq, qd, eps);
  const KVShape cache = cache_shape(bf, R, r, kc, vc);
  const int B = proj.size(0), S = proj.size(1), rows = (int)start + S;
  CHK((slots || B <= kc.size(0)) && rows <= cache.rows && B > 0 && S > 0);
  const Step step = make_step(slots, c10::nullopt, lens, start, false, B);
  auto qw = torch::empty({B, S, H, qd}, proj.options());
  auto lw = torch::empty({B, rows, R}, proj.options()), rw = torch::empty({B, rows, r}, proj.options());
  const hipStream_t stream = cur_stream();
  BY_TYPE(dt, {
    if (start > 0)
      hipLaunchKernelGGL((latent_history_kernel<T>), dim3(start, B), dim3(256), 0, stream, P<T>(kc), M<T>(lw), M<T>(rw),
                         cache, rows, (int)R, (int)r, step);
    hipLaunchKernelGGL((latent_append_kernel<T>), dim3(S, B), dim3(256), 0, stream, P<T>(proj), P<T>(norm),
                       freq.data_ptr<float>(), M<T>(qw), (T*)nullptr, (T*)nullptr, M<T>(kc), M<T>(vc), M<T>(lw),
                       M<T>(rw), cache, rows, (int)start, a, step);
  });
  return {qw, lw, rw};
}

// Decode: -> unrotated queries [H,B,d], rotated ones [B,H,r]
std::vector<Tensor> latent_append_step(Tensor proj, int64_t q_at, int64_t c_at, int64_t H, int64_t d, int64_t r,
                                       int64_t R, Tensor norm, Tensor freq, double eps, Tensor kc, Tensor vc,
                                       OptT slots, OptT positions) {
  const auto dt = io_type(proj);
  check_io(kc, dt);
  check_io(vc, dt);
  const LatArgs a = lat_args(proj, q_at, c_at, H, d, r, R, norm, freq, 0, eps);
  const KVShape cache = cache_shape(dt == torch::kBFloat16, R, r, kc, vc);
  const int B = proj.size(0);
  CHK((slots || B <= kc.size(0)) && B > 0 && proj.size(1) == 1);
  const Step step = make_step(slots, positions, c10::nullopt, 0, true, B);
  auto qn = torch::empty({H, B, d}, proj.options()), qr = torch::empty({B, H, r}, proj.options());
  BY_TYPE(dt, {
    hipLaunchKernelGGL((latent_append_kernel<T>), dim3(1, B), dim3(256), 0, cur_stream(), P<T>(proj), P<T>(norm),
                       freq.data_ptr<float>(), (T*)nullptr, M<T>(qn), M<T>(qr), M<T>(kc), M<T>(vc), (T*)nullptr,
                       (T*)nullptr, cache, 0, 0, a, step);
  });
  return {qn, qr};
}

// kv [B,rows,H*d + H*e], rot [B,rows,r] -> packed keys and values, and their rows
std::tuple<Tensor, Tensor, int64_t> pack_heads(Tensor kv, Tensor rot, int64_t H, int64_t d, int64_t r, int64_t e) {
  const auto dt = io_type(kv);
  const bool bf = dt == torch::kBFloat16;
  check_io(rot, dt);
  CHK(kv.dim() == 3 && rot.dim() == 3 && kv.size(2) == H * (d + e) && rot.size(2) == r && rot.size(0) == kv.size(0) &&
      rot.size(1) == kv.size(1) && H <= 65535 && kv.size(0) <= 65535);
  const int B = kv.size(0), rows = kv.size(1);
  KVShape ws{(int)(d + r), (int)e, (int)(d + r + 31) / 32, (int)(e + 15) / 16, bf ? (rows + 31) / 32 * 32 : rows, INT_MAX};
  auto kw = torch::empty({B, H, (int64_t)ws.rows * (bf ? ws.kc * 32 : ws.dim)}, kv.options());
  auto vw = torch::empty({B, H, (int64_t)ws.rows * (bf ? ws.vg * 16 : ws.vdim)}, kv.options());
  BY_TYPE(dt, {
    hipLaunchKernelGGL((pack_heads_kernel<T>), dim3((rows + 31) / 32, H, B), dim3(256), 0, cur_stream(), P<T>(kv),
                       P<T>(rot), M<T>(kw), M<T>(vw), ws, rows, (int)H, (int)d, (int)r, (int)e);
  });
  return {kw, vw, ws.rows};
}

// Folded queries ql [H,B,R] and rotated ones qr [B,H,r] against the cache:
// -> weighted latents [H,B,R]
Tensor latent_decode(Tensor ql, Tensor qr, Tensor kc, Tensor vc, double scale, OptT slots, Tensor positions,
                     OptT sinks) {
  const auto dt = io_type(ql);
  const bool bf = dt == torch::kBFloat16;
  for (const Tensor& t : {qr, kc, vc}) check_io(t, dt);
  CHK(ql.dim() == 3 && qr.dim() == 3 && qr.size(0) == ql.size(1) && qr.size(1) == ql.size(0));
  const int H = ql.size(0), B = ql.size(1), R = ql.size(2), r = qr.size(2);
  const KVShape cache = cache_shape(bf, R, r, kc, vc);
  CHK((slots || B <= kc.size(0)) && B > 0 && B <= 65535);
  if (sinks) { check_io(*sinks, dt); CHK(sinks->numel() == H); }
  const Step step = make_step(slots, positions, c10::nullopt, 0, true, B);
  auto out = torch::empty_like(ql);
  const hipStream_t stream = cur_stream();
  if (!bf) {
    const size_t lds = (2 * R + r) * sizeof(float);
    TORCH_CHECK(lds <= 60000, "a latent of ", R, " channels does not fit LDS");
    hipLaunchKernelGGL(latent_decode_f32_kernel, dim3(H, B), dim3(256), lds, stream, P<float>(ql), P<float>(qr),
                       P<float>(kc), P<float>(vc), sinks ? P<float>(*sinks) : nullptr, M<float>(out), cache,
                       (float)scale, H, R, r, step);
    return out;
  }
  const size_t lds = 16 * (cache.kc * 32 + 8) * sizeof(bf16_t);
  TORCH_CHECK(lds <= 56000 && cache.vg <= 64, "a latent of ", R, " channels does not fit LDS");
  const int hg = (H + 15) / 16;
  const int splits = std::max(1, std::min((512 + B * hg - 1) / (B * hg), cache.rows / 128));
  Tensor part;
  if (splits > 1) part = f32(ql, {B, splits, H, R + 2});
  float* pp = splits > 1 ? M<float>(part) : nullptr;
  const bf16_t* sp = sinks ? P<bf16_t>(*sinks) : nullptr;
  const dim3 grid(splits, hg, B);
#define DECODE(GW)                                                                                                \
  hipLaunchKernelGGL((latent_decode_kernel<GW>), grid, dim3(256), lds, stream, P<bf16_t>(ql), P<bf16_t>(qr),      \
                     P<bf16_t>(kc), P<bf16_t>(vc), sp, M<bf16_t>(out), pp, splits, cache, (float)scale, H, R, r, step)
  const int gw = (cache.vg + 3) / 4;
  if (gw <= 2) DECODE(2);
  else if (gw <= 4) DECODE(4);
  else if (gw <= 8) DECODE(8);
  else DECODE(16);
#undef DECODE
  if (splits > 1)
    hipLaunchKernelGGL(latent_merge_kernel, dim3(H, B), dim3(256), splits * sizeof(float), stream, pp, sp, M<bf16_t>(out), splits, H, R, step);
  return out;
}

void gather_heads(Tensor o, OptT gates, int64_t g_at, Tensor out, int64_t out_at, double out_scale) {
  const auto dt = io_type(o);
  check_io(out, dt);
  CHK(o.dim() == 3 && out.dim() == 3 && out.size(0) == o.size(1) && out.size(1) == 1);
  const int H = o.size(0), B = o.size(1), e = o.size(2), K = out.size(2), N = gates ? gates->size(2) : 0;
  CHK(out_at >= 0 && out_at + H * e <= K && B <= 65535);
  if (gates) {
    check_io(*gates, dt);
    CHK(gates->dim() == 3 && gates->size(0) == B && gates->size(1) == 1 && g_at >= 0 && g_at + H * e <= N);
  }
  if (B == 0) return;
#define GATHER(V)                                                                                                   \
  hipLaunchKernelGGL((gather_heads_kernel<T, V>), dim3((H * e + 256 * V - 1) / (256 * V), B), dim3(256), 0,         \
                     cur_stream(), P<T>(o), gates ? P<T>(*gates) : nullptr, M<T>(out), B, H * e, e, N, (int)g_at, K, \
                     (int)out_at, (float)out_scale)
  BY_TYPE(dt, {
    if (((e | N | g_at | K | out_at) & 3) == 0) GATHER(4);
    else GATHER(1);
  });
#undef GATHER
}

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.def("latent_append", &latent_append, "latent norm, rotations, cache append and workspaces of a prompt chunk");
  m.def("latent_append_step", &latent_append_step, "the same for a decode step");
  m.def("pack_heads", &pack_heads, "expanded keys and values of all heads in attention order");
  m.def("latent_decode", &latent_decode, "decode attention of all heads over cached latents, with sinks",
        py::arg("ql"), py::arg("qr"), py::arg("kc"), py::arg("vc"), py::arg("scale"), py::arg("slots"),
        py::arg("positions"), py::arg("sinks") = py::none());
  m.def("gather_heads", &gather_heads, "expanded outputs of a decode step by token, times their gates");
}
