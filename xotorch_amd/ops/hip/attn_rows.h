// Softmax attention over rows of a cache on CDNA4 (gfx950): one flash kernel
// for prompts and one split kernel for decode steps, in four modes:
//   WINDOW: sliding window, learned bias per distance bucket, a zero-score
//           sink, a sigmoid gate per head
//   CHUNK:  keys of the query's own chunk of the sequence, a bias that falls
//           linearly with the distance, a learned sink per head
//   CAUSAL: all earlier keys; a learned sink per head or none; a sigmoid gate per
//           value channel or none (prompts only)
//   KEPT:   sliding window (or none) that keeps the first tokens in sight,
//           capped scores, one or two maps over the same values, of which the
//           second is subtracted and the difference normed
//
// Two element types: bf16 (MFMA over fragment-packed keys and values) and fp32
// (plain layouts, plain fp32 arithmetic). Scores, softmax and norms are fp32
// in both. Rows address caches by slot (struct Step): slot -1 is a parked row.
#pragma once

#include "common.h"

struct AttnArgs {
  int S, H, G, N, K;                    // tokens a row, heads, projection and output widths
  int q_at, k_at, v_at, g_at, out_at;
  int qd;                               // padded dims of the q workspace
  float scale, eps, out_scale;
  int window, nb;                       // window or chunk length; entries of the distance table
  // KEPT: first tokens that stay in sight; whether prompts read the cache (rows
  // by slot) instead of a workspace; cap of the scores (0: none), norm's factor
  // and the second map's weight
  int keep, by_slot;
  float cap, gain;
  const float* lam;
};

enum Mode { WINDOW, CHUNK, CAUSAL, KEPT };

// Keys that position pos sees: itself and the reach - 1 before it.
template <int MODE>
DEVINL int reach_of(const AttnArgs& a, int pos) {
  return MODE == WINDOW || MODE == KEPT ? a.window : MODE == CHUNK ? pos % a.window + 1 : pos + 1;
}
// Slope of the linear distance bias: halves 8 times over the heads.
DEVINL float slope_of(const AttnArgs& a, int h) { return exp2f(-8.f * (float)(h + 1) / (float)a.H); }

// cap tanh(v / cap)
DEVINL float capped(float v, float cap) {
  const float e = __expf(2.f * v * __builtin_amdgcn_rcpf(cap));
  return cap * (1.f - 2.f * __builtin_amdgcn_rcpf(1.f + e));
}
// Row of position p: the first `keep` have their own, the others follow from
// position `base` on, in a ring of `mod`.
DEVINL int place_of(int p, int keep, int base, int mod) { return p < keep ? p : keep + (p - base) % mod; }

// What joins the softmax beside the keys, and what scales a head's output.
template <int MODE, typename T>
struct Side {
  const T *proj, *sinks;
  // score of the extra entry in the denominator
  DEVINL float sink(int h) const {
    return MODE == WINDOW ? 0.f : MODE == CHUNK || (MODE == CAUSAL && sinks) ? ld(sinks + h) : -INFINITY;
  }
  // where the running maximum starts: finite, so that fully masked tiles are harmless
  DEVINL float start(int h) const { return (MODE == CAUSAL && !sinks) || MODE == KEPT ? -1e30f : sink(h); }
  DEVINL float gate(const AttnArgs& a, size_t tok, int h) const {
    return MODE == WINDOW ? a.out_scale * sigmoidf(ld(proj + tok * a.N + a.g_at + h)) : a.out_scale;
  }
  // CAUSAL: columns of a token's gates, one per value channel of a head
  DEVINL const T* gates(const AttnArgs& a, size_t tok, int h, int vdim) const {
    return MODE == CAUSAL && proj ? proj + tok * a.N + a.g_at + h * vdim : nullptr;
  }
};

// Flash prefill on matrix cores: a wave owns 32 queries of one head and walks
// the key tiles that their windows touch. EXACT: kc == KC and vg == VG.
template <int KC, int VG, bool EXACT, int MODE, int MAPS = 1, int QT = 2>
__global__ __launch_bounds__(256) void attn_rows_prefill_kernel(
    const bf16_t* __restrict__ qw, const bf16_t* __restrict__ kw, const bf16_t* __restrict__ vw,
    Side<MODE, bf16_t> side, const int* __restrict__ bucket, const bf16_t* __restrict__ rel,
    bf16_t* __restrict__ out, KVShape ws, int hist, AttnArgs a, Step step) {
  extern __shared__ float bias[];  // [nb], this head's bias per distance
  const int h = blockIdx.y, b = blockIdx.z, g = h / (a.H / a.G);
  const int lane = threadIdx.x & 63, col = lane & 15, quad = lane >> 4;
  if (MODE == WINDOW) {
    for (int i = threadIdx.x; i < a.nb; i += 256) bias[i] = ld(rel + bucket[i] * a.H + h);
    __syncthreads();
  }
  const float slope = MODE == CHUNK ? slope_of(a, h) : 0.f, sink = side.sink(h);
  constexpr int NT = MAPS * QT;  // tiles of 16 queries: of the first map, then of the second
  const int s0 = (blockIdx.x * 4 + (threadIdx.x >> 6)) * QT * 16;
  if (s0 >= a.S) return;
  const int kc = EXACT ? KC : ws.kc, vg = EXACT ? VG : ws.vg;
  bf16x8 qf[NT][KC];
#pragma unroll
  for (int t = 0; t < NT; ++t) {
    const int s = min(s0 + t % QT * 16 + col, a.S - 1);
    const bf16_t* q = qw + ((((size_t)b * a.S + s) * a.H + h) * MAPS + t / QT) * a.qd + quad * 8;
#pragma unroll
    for (int c = 0; c < KC; ++c)
      if (EXACT || c < kc) qf[t][c] = *(const bf16x8*)(q + c * 32);
  }
  // the sink's score bounds the maximum from below
  float m[NT], l[NT];
  int reach[QT];
  floatx4 o[NT][VG];
#pragma unroll
  for (int t = 0; t < NT; ++t) {
    m[t] = side.start(h);
    l[t] = 0.f;
    if (t < QT) reach[t] = reach_of<MODE>(a, step.start + s0 + t * 16 + col);
#pragma unroll
    for (int i = 0; i < VG; ++i) o[t][i] = (floatx4)(0.f);
  }
  const size_t head = (size_t)(MODE == KEPT && a.by_slot ? max(step.slot(b), 0) : b) * a.G + g;
  const bf16_t* kb[MAPS];
#pragma unroll
  for (int mp = 0; mp < MAPS; ++mp) kb[mp] = kw + Layout<bf16_t>::kbase(ws, head * MAPS + mp);
  const bf16_t* vb = vw + Layout<bf16_t>::vbase(ws, head);
  const int vstride = (ws.rows >> 5) * 512;
  const int t0 = max(0, hist + s0 + 1 - reach_of<MODE>(a, step.start + s0)) >> 5;
  const int t1 = (hist + min(s0 + QT * 16 - 1, a.S - 1)) >> 5;
  const int kept = MODE == KEPT ? (a.keep + 31) >> 5 : 0;  // tiles of the first tokens
  // two maps leave room for one wave a SIMD: keys are loaded a tile ahead, values
  // before the softmax
  constexpr bool AHEAD = MAPS == 2 && KC <= 4;
  bf16x8 kf[2][MAPS][KC];
  auto load_keys = [&](int tile) {
#pragma unroll
    for (int hf = 0; hf < 2; ++hf)
#pragma unroll
      for (int c = 0; c < KC; ++c)
        if (EXACT || c < kc)
#pragma unroll
          for (int mp = 0; mp < MAPS; ++mp)
            kf[hf][mp][c] = *(const bf16x8*)(kb[mp] + ((size_t)(tile * 2 + hf) * kc + c) * 512 + lane * 8);
  };
  int next = kept ? 0 : t0;
  if (AHEAD) load_keys(next);
  while (next <= t1) {
    const int tile = next;
    if (!AHEAD) load_keys(tile);
    next = MODE == KEPT && tile + 1 >= kept && tile + 1 < t0 ? t0 : tile + 1;
    floatx4 sc[NT][2];
#pragma unroll
    for (int hf = 0; hf < 2; ++hf) {
#pragma unroll
      for (int t = 0; t < NT; ++t) sc[t][hf] = (floatx4)(0.f);
#pragma unroll
      for (int c = 0; c < KC; ++c)
        if (EXACT || c < kc)
#pragma unroll
          for (int mp = 0; mp < MAPS; ++mp)
#pragma unroll
            for (int t = mp * QT; t < mp * QT + QT; ++t)
              sc[t][hf] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[hf][mp][c], qf[t][c], sc[t][hf], 0, 0, 0);
    }
    bf16x8 vf[VG];
    auto load_value = [&](int i) { vf[i] = *(const bf16x8*)(vb + (size_t)i * vstride + (size_t)tile * 512 + lane * 8); };
    if (AHEAD) {
#pragma unroll
      for (int i = 0; i < VG; ++i)
        if (EXACT || i < vg) load_value(i);
      load_keys(min(next, t1));
      __builtin_amdgcn_sched_barrier(0);
    }
    bf16x8 pf[NT];
#pragma unroll
    for (int t = 0; t < NT; ++t) {
      // distance to this lane's first key of the tile
      const int dist0 = hist + s0 + t % QT * 16 + col - tile * 32 - quad * 4;
      float top = m[t];
#pragma unroll
      for (int hf = 0; hf < 2; ++hf)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int dist = dist0 - hf * 16 - r;
          float v = sc[t][hf][r] * a.scale;
          if (MODE == WINDOW) v += bias[min(max(dist, 0), a.nb - 1)];
          if (MODE == CHUNK) v -= slope * (float)dist;
          if (MODE == KEPT && a.cap != 0.f) v = capped(v, a.cap);
          const bool first = MODE == KEPT && tile * 32 + quad * 4 + hf * 16 + r < a.keep;
          sc[t][hf][r] = (dist >= 0 && (dist < reach[t % QT] || first)) ? v : -INFINITY;
          top = fmaxf(top, sc[t][hf][r]);
        }
      top = fmaxf(top, __shfl_xor(top, 16));
      top = fmaxf(top, __shfl_xor(top, 32));
      if (__any(top > m[t])) {
        const float al = __expf(m[t] - top);
        m[t] = top;
        l[t] *= al;
#pragma unroll
        for (int i = 0; i < VG; ++i) o[t][i] *= al;
      }
      float sum = 0.f;
#pragma unroll
      for (int hf = 0; hf < 2; ++hf)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const float p = __expf(sc[t][hf][r] - top);
          sum += p;
          pf[t][hf * 4 + r] = (__bf16)p;
        }
      l[t] += sum;
    }
#pragma unroll
    for (int i = 0; i < VG; ++i)
      if (EXACT || i < vg) {
        if (!AHEAD) load_value(i);
#pragma unroll
        for (int t = 0; t < NT; ++t) o[t][i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf[i], pf[t], o[t][i], 0, 0, 0);
      }
  }
  const int len = step.slot(b) < 0 ? 0 : step.len(b, a.S);
#pragma unroll
  for (int t = 0; t < QT; ++t) {
    const int s = s0 + t * 16 + col;
    float sum = l[t];
    sum += __shfl_xor(sum, 16);
    sum += __shfl_xor(sum, 32);
    float f = 0.f;
    if (MAPS == 2) {  // difference of the maps, normed
      float sum2 = l[NT - QT + t], ss = 0.f;
      sum2 += __shfl_xor(sum2, 16);
      sum2 += __shfl_xor(sum2, 32);
      const float f1 = 1.f / sum, f2 = *a.lam / sum2;
#pragma unroll
      for (int i = 0; i < VG; ++i)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const float d = o[t][i][r] * f1 - o[NT - QT + t][i][r] * f2;
          o[t][i][r] = d;
          ss += d * d;
        }
      ss += __shfl_xor(ss, 16);
      ss += __shfl_xor(ss, 32);
      f = a.gain / sqrtf(ss / (float)ws.vdim + a.eps);
    }
    if (s >= a.S) continue;
    const size_t tok = (size_t)b * a.S + s;
    if (s < len) f = side.gate(a, tok, h) * (MAPS == 2 ? f : 1.f / (sum + __expf(sink - m[t])));
    bf16_t* dst = out + tok * a.K + a.out_at + h * ws.vdim;
    if (const bf16_t* gate = side.gates(a, tok, h, ws.vdim)) {
      const bool vec = ((a.N | a.g_at | ws.vdim) & 3) == 0;
#pragma unroll
      for (int i = 0; i < VG; ++i) {
        const int c = i * 16 + quad * 4;
        float g[4];
        if (vec && c < ws.vdim) ld4(gate + c, g);
        else
#pragma unroll
          for (int r = 0; r < 4; ++r) g[r] = c + r < ws.vdim ? ld(gate + c + r) : 0.f;
#pragma unroll
        for (int r = 0; r < 4; ++r) o[t][i][r] *= sigmoidf(g[r]);
      }
    }
#pragma unroll
    for (int i = 0; i < VG; ++i) {
      const int c = i * 16 + quad * 4;
      if (c + 3 < ws.vdim && (ws.vdim & 3) == 0) {
        float v[4];
#pragma unroll
        for (int r = 0; r < 4; ++r) v[r] = s < len ? o[t][i][r] * f : 0.f;
        st4(dst + c, v);
      } else {
#pragma unroll
        for (int r = 0; r < 4; ++r)
          if (c + r < ws.vdim) st(dst + c + r, s < len ? o[t][i][r] * f : 0.f);
      }
    }
  }
}

// Split decode: a block scores one row's ring (or a part of it) for up to 16
// query heads of a kv head; its 4 waves walk 32-row tiles and merge in LDS.
// part null: the block saw the whole ring and writes the result.
template <int KC, int VG, bool EXACT, int MODE, int MAPS = 1>
__global__ __launch_bounds__(256) void attn_rows_decode_kernel(
    const bf16_t* __restrict__ qw, const bf16_t* __restrict__ kc_, const bf16_t* __restrict__ vc_,
    Side<MODE, bf16_t> side, const int* __restrict__ bucket, const bf16_t* __restrict__ rel, int rel_rows,
    bf16_t* __restrict__ out, float* __restrict__ part, int splits, KVShape ring, AttnArgs a, Step step) {
  constexpr int OW = VG * 16 + 4;  // row of a wave's partial output (padded)
  __shared__ float po[4][16 * OW];
  __shared__ float pm[4][16], pl[4][16];
  __shared__ float diff[MAPS == 2 ? 16 * OW : 1];
  extern __shared__ int tab[];  // [nb] buckets, then [rel_rows][16] bias of these heads
  const int split = blockIdx.x, b = blockIdx.z;
  const int per = a.H / a.G, qgs = (per + 15) >> 4;
  const int g = blockIdx.y / qgs, q0 = (blockIdx.y % qgs) * 16, nq = min(16, per - q0);
  const int h0 = g * per + q0;
  const int slot = step.slot(b);
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, col = lane & 15, quad = lane >> 4;
  if (slot < 0) {
    if (!part)
      for (int i = threadIdx.x; i < nq * ring.vdim; i += 256)
        st(out + (size_t)b * a.K + a.out_at + (size_t)h0 * ring.vdim + i, 0.f);
    return;
  }
  float* relb = (float*)(tab + a.nb);
  if (MODE == WINDOW) {
    for (int i = threadIdx.x; i < a.nb; i += 256) tab[i] = bucket[i];
    for (int i = threadIdx.x; i < rel_rows * 16; i += 256)
      relb[i] = (i & 15) < nq ? ld(rel + (i >> 4) * a.H + h0 + (i & 15)) : 0.f;
    __syncthreads();
  }
  const int hc = h0 + min(col, nq - 1);  // this lane's head
  const float slope = MODE == CHUNK ? slope_of(a, hc) : 0.f;
  const int kc = EXACT ? KC : ring.kc, vg = EXACT ? VG : ring.vg;
  const int pos = step.first(b), cur = MODE == KEPT ? place_of(pos, a.keep, a.keep, ring.mod) : pos % ring.mod;
  // CHUNK: rows past the current one still hold an earlier chunk
  const int seen = MODE == CHUNK ? min(cur + 1, ring.rows) : min(min(a.window, ring.rows), pos + 1);
  const int ntiles = ((MODE == CHUNK ? seen : min(ring.rows, pos + 1)) + 31) >> 5;
  const int per_split = (ntiles + splits - 1) / splits;
  bf16x8 qf[MAPS][KC];
  float m[MAPS], l[MAPS];
  floatx4 o[MAPS][VG];
  const bf16_t* kb[MAPS];
#pragma unroll
  for (int mp = 0; mp < MAPS; ++mp) {
    const bf16_t* q = qw + (((size_t)b * a.H + hc) * MAPS + mp) * a.qd + quad * 8;
#pragma unroll
    for (int c = 0; c < KC; ++c)
      if (EXACT || c < kc) qf[mp][c] = *(const bf16x8*)(q + c * 32);
    m[mp] = side.start(hc);
    l[mp] = 0.f;
#pragma unroll
    for (int i = 0; i < VG; ++i) o[mp][i] = (floatx4)(0.f);
    kb[mp] = kc_ + Layout<bf16_t>::kbase(ring, ((size_t)slot * a.G + g) * MAPS + mp);
  }
  const bf16_t* vb = vc_ + Layout<bf16_t>::vbase(ring, (size_t)slot * a.G + g);
  const size_t vstride = (size_t)(ring.rows >> 5) * 512;
  const int end = min(ntiles, (split + 1) * per_split);
  for (int tile = split * per_split + wave; tile < end; tile += 4) {
    bf16x8 vf[VG];
    floatx4 sc[MAPS][2];
#pragma unroll
    for (int mp = 0; mp < MAPS; ++mp)
#pragma unroll
      for (int hf = 0; hf < 2; ++hf) {
        sc[mp][hf] = (floatx4)(0.f);
#pragma unroll
        for (int c = 0; c < KC; ++c)
          if (EXACT || c < kc) {
            const bf16x8 kf = *(const bf16x8*)(kb[mp] + ((size_t)(tile * 2 + hf) * kc + c) * 512 + lane * 8);
            sc[mp][hf] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf[mp][c], sc[mp][hf], 0, 0, 0);
          }
      }
#pragma unroll
    for (int i = 0; i < VG; ++i)
      if (EXACT || i < vg) vf[i] = *(const bf16x8*)(vb + i * vstride + (size_t)tile * 512 + lane * 8);
#pragma unroll
    for (int mp = 0; mp < MAPS; ++mp) {
      float top = m[mp];
#pragma unroll
      for (int hf = 0; hf < 2; ++hf)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int row = tile * 32 + hf * 16 + quad * 4 + r;
          int age = cur - row;
          if (age < 0) age += MODE == KEPT ? ring.mod : ring.rows;
          float v = sc[mp][hf][r] * a.scale;
          if (MODE == WINDOW) v += relb[tab[min(age, a.nb - 1)] * 16 + col];
          if (MODE == CHUNK) v -= slope * (float)age;
          if (MODE == KEPT && a.cap != 0.f) v = capped(v, a.cap);
          // KEPT: the first rows are the first tokens'; of the others, those that
          // hold a token of the window
          const bool on = MODE != KEPT ? age < seen : row < a.keep ? row <= pos : age < a.window && pos - age >= a.keep;
          sc[mp][hf][r] = on ? v : -INFINITY;
          top = fmaxf(top, sc[mp][hf][r]);
        }
      top = fmaxf(top, __shfl_xor(top, 16));
      top = fmaxf(top, __shfl_xor(top, 32));
      const float al = __expf(m[mp] - top);
      m[mp] = top;
      l[mp] *= al;
      bf16x8 pf;
#pragma unroll
      for (int hf = 0; hf < 2; ++hf)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const float p = __expf(sc[mp][hf][r] - top);
          l[mp] += p;
          pf[hf * 4 + r] = (__bf16)p;
        }
#pragma unroll
      for (int i = 0; i < VG; ++i)
        if (EXACT || i < vg) {
          o[mp][i] *= al;
          o[mp][i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf[i], pf, o[mp][i], 0, 0, 0);
        }
    }
  }
#pragma unroll
  for (int mp = 0; mp < MAPS; ++mp) {
    l[mp] += __shfl_xor(l[mp], 16);
    l[mp] += __shfl_xor(l[mp], 32);
    if (mp) __syncthreads();
    if (quad == 0) { pm[wave][col] = m[mp]; pl[wave][col] = l[mp]; }
#pragma unroll
    for (int i = 0; i < VG; ++i)
#pragma unroll
      for (int r = 0; r < 4; ++r) po[wave][col * OW + i * 16 + quad * 4 + r] = o[mp][i][r];
    __syncthreads();
    for (int i = threadIdx.x; i < nq * ring.vdim; i += 256) {
      const int qh = i / ring.vdim, c = i - qh * ring.vdim;
      const int h = h0 + qh;
      float M = side.start(h), L = 0.f, O = 0.f;
#pragma unroll
      for (int w = 0; w < 4; ++w) M = fmaxf(M, pm[w][qh]);
#pragma unroll
      for (int w = 0; w < 4; ++w) {
        const float f = __expf(pm[w][qh] - M);
        L += f * pl[w][qh];
        O += f * po[w][qh * OW + c];
      }
      if (part) {
        float* p = part + ((((size_t)b * splits + split) * a.H + h) * MAPS + mp) * (ring.vdim + 2);
        p[2 + c] = O;
        if (c == 0) { p[0] = M; p[1] = L; }
      } else if (MAPS == 2) {
        if (mp == 0) diff[qh * OW + c] = O / L;
        else diff[qh * OW + c] -= *a.lam * O / L;
      } else {
        st(out + (size_t)b * a.K + a.out_at + (size_t)h * ring.vdim + c,
           O / (L + __expf(side.sink(h) - M)) * side.gate(a, b, h));
      }
    }
  }
  if (MAPS == 1 || part) return;
  __syncthreads();
  for (int qh = wave; qh < nq; qh += 4) {
    float ss = 0.f;
    for (int c = lane; c < ring.vdim; c += 64) ss += diff[qh * OW + c] * diff[qh * OW + c];
    const float f = a.gain / sqrtf(wave_sum(ss) / (float)ring.vdim + a.eps) * side.gate(a, b, h0 + qh);
    for (int c = lane; c < ring.vdim; c += 64)
      st(out + (size_t)b * a.K + a.out_at + (size_t)(h0 + qh) * ring.vdim + c, diff[qh * OW + c] * f);
  }
}

// Partial results of a head's splits -> its output. Four waves take splits in
// turn, a few in flight; then a thread has a value column.
template <int MODE, int MAPS = 1>
__global__ __launch_bounds__(256) void attn_rows_merge_kernel(
    const float* __restrict__ part, Side<MODE, bf16_t> side, bf16_t* __restrict__ out, int splits,
    int vdim, AttnArgs a, Step step) {
  constexpr int NC = 4, AHEAD = 4;  // value columns of a lane; splits in flight
  __shared__ float po[MAPS][4][NC * 64], pm[MAPS][4], pl[MAPS][4], sums[4];
  const int h = blockIdx.x, b = blockIdx.y, wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int c = threadIdx.x;
  float v = 0.f;
  if (step.slot(b) >= 0) {
    float M[MAPS], L[MAPS], O[MAPS][NC];
#pragma unroll
    for (int mp = 0; mp < MAPS; ++mp) {
      M[mp] = side.start(h);
      L[mp] = 0.f;
#pragma unroll
      for (int i = 0; i < NC; ++i) O[mp][i] = 0.f;
    }
    for (int s0 = wave; s0 < splits; s0 += 4 * AHEAD) {
      float m[MAPS][AHEAD], l[MAPS][AHEAD], o[MAPS][AHEAD][NC];
#pragma unroll
      for (int mp = 0; mp < MAPS; ++mp)
#pragma unroll
        for (int j = 0; j < AHEAD; ++j) {
          const int s = s0 + 4 * j;
          const float* p = part + ((((size_t)b * splits + min(s, splits - 1)) * a.H + h) * MAPS + mp) * (vdim + 2);
          m[mp][j] = s < splits ? p[0] : -INFINITY;
          l[mp][j] = p[1];
#pragma unroll
          for (int i = 0; i < NC; ++i) o[mp][j][i] = p[2 + min(lane + i * 64, vdim - 1)];
        }
#pragma unroll
      for (int mp = 0; mp < MAPS; ++mp) {
        float top = M[mp];
#pragma unroll
        for (int j = 0; j < AHEAD; ++j) top = fmaxf(top, m[mp][j]);
        const float al = __expf(M[mp] - top);
        M[mp] = top;
        L[mp] *= al;
#pragma unroll
        for (int i = 0; i < NC; ++i) O[mp][i] *= al;
#pragma unroll
        for (int j = 0; j < AHEAD; ++j) {
          const float f = __expf(m[mp][j] - top);
          L[mp] += f * l[mp][j];
#pragma unroll
          for (int i = 0; i < NC; ++i) O[mp][i] += f * o[mp][j][i];
        }
      }
    }
#pragma unroll
    for (int mp = 0; mp < MAPS; ++mp) {
#pragma unroll
      for (int i = 0; i < NC; ++i) po[mp][wave][i * 64 + lane] = O[mp][i];
      if (lane == 0) { pm[mp][wave] = M[mp]; pl[mp][wave] = L[mp]; }
    }
    __syncthreads();
#pragma unroll
    for (int mp = 0; mp < MAPS; ++mp) {
      float top = pm[mp][0], sum = 0.f, all = 0.f;
#pragma unroll
      for (int w = 1; w < 4; ++w) top = fmaxf(top, pm[mp][w]);
#pragma unroll
      for (int w = 0; w < 4; ++w) {
        const float f = __expf(pm[mp][w] - top);
        all += f * pl[mp][w];
        sum += f * po[mp][w][c];
      }
      v += sum * (MAPS == 1 ? side.gate(a, b, h) / (all + __expf(side.sink(h) - top)) : mp ? -*a.lam / all : 1.f / all);
    }
  }
  if (MAPS == 2) {
    const float ss = wave_sum(c < vdim ? v * v : 0.f);
    if (lane == 0) sums[wave] = ss;
    __syncthreads();
    v *= a.gain / sqrtf((sums[0] + sums[1] + sums[2] + sums[3]) / (float)vdim + a.eps) * side.gate(a, b, h);
  }
  if (c < vdim) st(out + (size_t)b * a.K + a.out_at + (size_t)h * vdim + c, v);
}

// 32-bit attention, one wave per (token, head): lanes over keys for the
// scores, over value columns for the sum. base/rows: where position p lies
// ((p - base) % mod, KEPT: place_of), so one kernel serves caches and
// workspaces. NC: value columns per lane.
template <int MODE, int NC, int MAPS = 1>
__global__ __launch_bounds__(64) void attn_rows_f32_kernel(
    const float* __restrict__ qw, const float* __restrict__ k, const float* __restrict__ v,
    Side<MODE, float> side, const int* __restrict__ bucket, const float* __restrict__ rel,
    float* __restrict__ out, KVShape kv, int base, AttnArgs a, Step step) {
  extern __shared__ float q[];  // [dim]
  const int s = blockIdx.x, h = blockIdx.y, b = blockIdx.z, g = h / (a.H / a.G), lane = threadIdx.x;
  const int slot = step.slot(b), len = step.decode ? 1 : step.len(b, a.S);
  float* dst = out + ((size_t)b * a.S + s) * a.K + a.out_at + (size_t)h * kv.vdim;
  if (slot < 0 || s >= len) {
    for (int c = lane; c < kv.vdim; c += 64) dst[c] = 0.f;
    return;
  }
  const size_t head = (size_t)(step.decode || (MODE == KEPT && a.by_slot) ? slot : b) * a.G + g;
  const float* vb = v + Layout<float>::vbase(kv, head);
  const int pos = min(step.first(b) + s, MODE == CAUSAL ? kv.rows - 1 : INT_MAX);
  const int lo = max(0, pos - reach_of<MODE>(a, pos) + 1);
  // keys in sight: the first tokens before the window, then the window
  const int early = MODE == KEPT ? min(a.keep, lo) : 0, count = early + pos - lo + 1;
  auto row_of = [&](int i) {
    const int p = i < early ? i : lo + i - early;
    return min(MODE == KEPT ? place_of(p, a.keep, base, kv.mod) : (p - base) % kv.mod, kv.rows - 1);
  };
  const float slope = MODE == CHUNK ? slope_of(a, h) : 0.f;
  float sum[NC], f = 0.f;
#pragma unroll
  for (int mp = 0; mp < MAPS; ++mp) {
    if (mp) __syncthreads();
    for (int d = lane; d < kv.dim; d += 64) q[d] = qw[((((size_t)b * a.S + s) * a.H + h) * MAPS + mp) * a.qd + d];
    __syncthreads();
    const float* kb = k + Layout<float>::kbase(kv, head * MAPS + mp);
    float m = side.start(h), l = 0.f, acc[NC];
#pragma unroll
    for (int i = 0; i < NC; ++i) acc[i] = 0.f;
    for (int i0 = 0; i0 < count; i0 += 64) {
      float sc = -INFINITY;
      if (i0 + lane < count) {
        const float* row = kb + Layout<float>::k(kv, row_of(i0 + lane), 0);
        const int dist = count - 1 - i0 - lane;
        float dot = 0.f;
        for (int d = 0; d < kv.dim; ++d) dot += q[d] * row[d];
        sc = dot * a.scale;
        if (MODE == WINDOW) sc += rel[bucket[min(dist, a.nb - 1)] * a.H + h];
        if (MODE == CHUNK) sc -= slope * (float)dist;
        if (MODE == KEPT && a.cap != 0.f) sc = a.cap * tanhf(sc / a.cap);
      }
      float top = sc;
#pragma unroll
      for (int x = 32; x > 0; x >>= 1) top = fmaxf(top, __shfl_xor(top, x));
      top = fmaxf(top, m);
      const float al = expf(m - top), e = expf(sc - top);
      m = top;
      l = l * al + wave_sum(e);
#pragma unroll
      for (int i = 0; i < NC; ++i) acc[i] *= al;
      const int n = min(64, count - i0);
      for (int j = 0; j < n; ++j) {
        const float pj = __shfl(e, j);
        const float* row = vb + Layout<float>::v(kv, row_of(i0 + j), 0);
#pragma unroll
        for (int i = 0; i < NC; ++i)
          if (lane + i * 64 < kv.vdim) acc[i] += pj * row[lane + i * 64];
      }
    }
    if (MAPS == 1) f = side.gate(a, (size_t)b * a.S + s, h) / (l + expf(side.sink(h) - m));
    else f = mp ? -*a.lam / l : 1.f / l;
#pragma unroll
    for (int i = 0; i < NC; ++i) sum[i] = mp ? sum[i] + acc[i] * f : acc[i] * f;
  }
  if (MAPS == 2) {
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < NC; ++i) ss += lane + i * 64 < kv.vdim ? sum[i] * sum[i] : 0.f;
    f = a.gain / sqrtf(wave_sum(ss) / (float)kv.vdim + a.eps) * side.gate(a, (size_t)b * a.S + s, h);
#pragma unroll
    for (int i = 0; i < NC; ++i) sum[i] *= f;
  }
  const float* gate = side.gates(a, (size_t)b * a.S + s, h, kv.vdim);
#pragma unroll
  for (int i = 0; i < NC; ++i)
    if (lane + i * 64 < kv.vdim) dst[lane + i * 64] = gate ? sum[i] / (1.f + expf(-gate[lane + i * 64])) : sum[i];
}

// ===========================================================================
// host side
// ===========================================================================

// template sizes: the smallest that hold both dims
#define BY_DIMS(kc, vg, RUN)                                           \
  if (kc <= 1 && vg <= 2) RUN(1, 2, (kc == 1 && vg == 2))              \
  else if (kc <= 2 && vg <= 4) RUN(2, 4, (kc == 2 && vg == 4))         \
  else if (kc <= 4 && vg <= 8) RUN(4, 8, (kc == 4 && vg == 8))         \
  else if (kc <= 6 && vg <= 8) RUN(6, 8, (kc == 6 && vg == 8))         \
  else RUN(8, 16, (kc == 8 && vg == 16))

// for two maps, whose values are usually twice as wide as a map's keys
#define BY_DIMS_2(kc, vg, RUN)                                         \
  if (kc <= 1 && vg <= 4) RUN(1, 4, (kc == 1 && vg == 4))              \
  else if (kc <= 2 && vg <= 8) RUN(2, 8, (kc == 2 && vg == 8))         \
  else if (kc <= 4 && vg <= 16) RUN(4, 16, (kc == 4 && vg == 16))      \
  else RUN(8, 16, (kc == 8 && vg == 16))

// Prompt rows [B,S,H,qd] against workspaces of rows [0, hist + S).
template <int MODE, int MAPS = 1>
static inline void prefill_rows(bool bf, int B, const Tensor& qw, const Tensor& kw, const Tensor& vw, const void* proj,
                         const void* sinks, const int* bucket, const void* rel, Tensor& out, const KVShape& ws,
                         int hist, int base, const AttnArgs& a, const Step& step) {
  const hipStream_t stream = cur_stream();
  TORCH_CHECK(B <= 65535 && a.H <= 65535, "a prefill step of ", B, " rows and ", a.H, " heads is too large");
  if (!bf) {
    const Side<MODE, float> side{(const float*)proj, (const float*)sinks};
    CHK(ws.vdim <= 256);
    hipLaunchKernelGGL((attn_rows_f32_kernel<MODE, 4, MAPS>), dim3(a.S, a.H, B), dim3(64), ws.dim * sizeof(float), stream,
                       P<float>(qw), P<float>(kw), P<float>(vw), side, bucket, (const float*)rel, M<float>(out), ws,
                       base, a, step);
    return;
  }
  const Side<MODE, bf16_t> side{(const bf16_t*)proj, (const bf16_t*)sinks};
  const size_t lds = MODE == WINDOW ? (size_t)a.nb * 4 : 0;
  TORCH_CHECK(lds <= 60000, "distance table of ", a.nb, " entries does not fit LDS");
#define RUN_QT(KC, VG, EXACT, QT)                                                                                    \
  hipLaunchKernelGGL((attn_rows_prefill_kernel<KC, VG, EXACT, MODE, MAPS, QT>),                                      \
                     dim3((a.S + QT * 64 - 1) / (QT * 64), a.H, B), dim3(256), lds, stream, P<bf16_t>(qw),           \
                     P<bf16_t>(kw), P<bf16_t>(vw), side, bucket, (const bf16_t*)rel, M<bf16_t>(out), ws, hist, a, step)
#define RUN(KC, VG, EXACT)                                                                                           \
  {                                                                                                                  \
    constexpr int QT = MAPS == 2 && VG > 8 ? 1 : 2; /* queries that the registers hold */                            \
    if (EXACT) RUN_QT(KC, VG, true, QT);                                                                             \
    else RUN_QT(KC, VG, false, QT);                                                                                  \
  }
  if constexpr (MAPS == 2) { BY_DIMS_2(ws.kc, ws.vg, RUN) }
  else { BY_DIMS(ws.kc, ws.vg, RUN) }
#undef RUN
#undef RUN_QT
}

// One token a row [B,1,H,qd] against the cache.
template <int MODE, int MAPS = 1>
static inline void decode_rows(bool bf, int B, const Tensor& qw, const Tensor& kc, const Tensor& vc, const void* proj,
                        const void* sinks, const int* bucket, const void* rel, int rel_rows, Tensor& out,
                        const KVShape& ring, int base, const AttnArgs& a, const Step& step) {
  const hipStream_t stream = cur_stream();
  if (!bf) {
    const Side<MODE, float> side{(const float*)proj, (const float*)sinks};
    hipLaunchKernelGGL((attn_rows_f32_kernel<MODE, 4, MAPS>), dim3(1, a.H, B), dim3(64), ring.dim * sizeof(float), stream,
                       P<float>(qw), P<float>(kc), P<float>(vc), side, bucket, (const float*)rel, M<float>(out), ring,
                       base, a, step);
    return;
  }
  const Side<MODE, bf16_t> side{(const bf16_t*)proj, (const bf16_t*)sinks};
  const size_t lds = MODE == WINDOW ? (size_t)a.nb * 4 + (size_t)rel_rows * 64 : 0;
  TORCH_CHECK(lds <= 60000, "distance table of ", a.nb, " entries does not fit LDS");
  const int qgs = (a.H / a.G + 15) / 16;
  // enough blocks for the chip, at least one 32-row tile per wave
  const int blocks = B * a.G * qgs;
  const int splits = std::max(1, std::min((512 + blocks - 1) / blocks, ring.rows / 128));
  Tensor part;
  if (splits > 1) part = f32(qw, {B, splits, a.H * MAPS, ring.vdim + 2});
  float* pp = splits > 1 ? M<float>(part) : nullptr;
  const dim3 grid(splits, a.G * qgs, B);
#define RUN(KC, VG, EXACT)                                                                                          \
  {                                                                                                                 \
    if (EXACT)                                                                                                      \
      hipLaunchKernelGGL((attn_rows_decode_kernel<KC, VG, true, MODE, MAPS>), grid, dim3(256), lds, stream, P<bf16_t>(qw), \
                         P<bf16_t>(kc), P<bf16_t>(vc), side, bucket, (const bf16_t*)rel, rel_rows, M<bf16_t>(out), pp, \
                         splits, ring, a, step);                                                                    \
    else                                                                                                            \
      hipLaunchKernelGGL((attn_rows_decode_kernel<KC, VG, false, MODE, MAPS>), grid, dim3(256), lds, stream, P<bf16_t>(qw), \
                         P<bf16_t>(kc), P<bf16_t>(vc), side, bucket, (const bf16_t*)rel, rel_rows, M<bf16_t>(out), pp, \
                         splits, ring, a, step);                                                                    \
  }
  if constexpr (MAPS == 2) { BY_DIMS_2(ring.kc, ring.vg, RUN) }
  else { BY_DIMS(ring.kc, ring.vg, RUN) }
#undef RUN
  if (splits > 1)
    hipLaunchKernelGGL((attn_rows_merge_kernel<MODE, MAPS>), dim3(a.H, B), dim3(256), 0, stream, pp, side, M<bf16_t>(out),
                       splits, ring.vdim, a, step);
}

static inline KVShape cache_shape(bool bf, int64_t G, int64_t dim, int64_t vdim, const Tensor& kc, const Tensor& vc,
                           int maps = 1) {
  KVShape ring{(int)dim, (int)vdim, (int)(dim + 31) / 32, (int)(vdim + 15) / 16, 0, 0};
  CHK(kc.size(1) == G * maps && vc.size(1) == G && kc.size(0) == vc.size(0));
  if (bf) {
    CHK(kc.dim() == 6 && vc.dim() == 6 && kc.size(3) == ring.kc && vc.size(2) == ring.vg);
    ring.rows = kc.size(2) * 16;
    CHK(ring.rows % 32 == 0 && vc.size(3) * 32 == ring.rows);
  } else {
    CHK(kc.dim() == 4 && vc.dim() == 4 && kc.size(3) == dim && vc.size(3) == vdim && kc.size(2) == vc.size(2));
    ring.rows = kc.size(2);
  }
  CHK(ring.rows > 0);
  ring.mod = ring.rows;
  return ring;
}

// One linear workspace of keys and values for a prompt chunk: `hist` earlier
// rows, then the chunk, padded to whole tiles.
struct Workspace {
  KVShape shape;
  Tensor k, v;
  int fill;
  Workspace(bool bf, const KVShape& ring, const Tensor& like, int B, int G, int hist, int S, int maps = 1)
      : shape(ring) {
    shape.rows = (hist + S + 31) / 32 * 32;
    shape.mod = INT_MAX;
    fill = shape.rows - hist;
    k = torch::empty({B, G * maps, (int64_t)shape.rows * (bf ? shape.kc * 32 : shape.dim)}, like.options());
    v = torch::empty({B, G, (int64_t)shape.rows * (bf ? shape.vg * 16 : shape.vdim)}, like.options());
  }
};
