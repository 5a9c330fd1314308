// CDNA4 (gfx950) kernels of sparse feed-forwards: a mixture of small experts,
// routed and computed without the host seeing a count.
//   - router: logits on matrix cores (fp32 accumulation), sigmoid scores, a
//     correction that only chooses, group-limited top-k, or a softmax over the
//     chosen logits; experts that every token uses, gated or not; counts per block
//   - place: every (token, expert) pair gets a row; rows of an expert lie
//     together, in token order
//   - grouped products: gate and up of a pair's token with the gated activation
//     in the epilogue, or up alone, squared where it is positive, then down; a
//     weight-streaming form for few tokens per expert and a tiled form for many.
//     A weight that multiplies a pair's input scales the product's rows
//   - add_norm: stream += mult * (a sublayer's output, or the weighted sum of a
//     token's expert rows), then the stream's norm for the next sublayer
//
// Two element types: bf16 and fp32 (fp32 MFMA throughout).

#include "common.h"

// ---------------------------------------------------------------------------
// router
// ---------------------------------------------------------------------------

constexpr int RT = 16;          // tokens of a router block
constexpr int MAX_EXPERTS = 512, MAX_PICK = 16;  // shared ones among the experts

// pick of E experts are chosen, then come top - pick that every token uses, all
// in all; tile: rows of a tile
// gate: the weight of these is the sigmoid of one more row of w, else one
struct RouteArgs { int T, D, E, top, groups, keep, nblk, tile; float scale; int pick, all, softmax, gate; };

// RW waves share k. Sixteen lanes choose for a token, J experts each.
template <typename T, bool WHOLE, int J, int RW>
__global__ __launch_bounds__(64 * RW) void route_kernel(
    const T* __restrict__ x, const T* __restrict__ w, const T* __restrict__ correction, int* __restrict__ idx,
    float* __restrict__ weight, int* __restrict__ rank, int* __restrict__ counts, RouteArgs a) {
  typedef Frag<T> F;
  extern __shared__ float lds[];  // choice, scores [RT][E]; partial sums [RW][RT][65]; chosen [RT][top]; open [RT]
  float* choice = lds;
  float* score = choice + RT * a.E;
  float* part = score + RT * a.E;
  int* chosen = (int*)(part + RW * RT * 65);
  float* open = (float*)(chosen + RT * a.top);  // [RT], the gate of the experts that every token uses
  const int Z = a.E + a.gate;
  const int t0 = blockIdx.x * RT, wave = threadIdx.x >> 6, lane = threadIdx.x & 63, col = lane & 15, quad = lane >> 4;
  const T* xr = x + (size_t)min(t0 + col, a.T - 1) * a.D;
  const int steps = (a.D + F::K - 1) / F::K;
  for (int e0 = 0; e0 < Z; e0 += 64) {
    floatx4 acc[4];
    const T* wr[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      acc[i] = (floatx4)(0.f);
      wr[i] = w + (size_t)min(e0 + i * 16 + col, Z - 1) * a.D;
    }
    auto run = [&](int c, auto count) {  // `count` steps from c on, loads first
      constexpr int UN = decltype(count)::value;
      typename F::V xf[UN], wf[UN][4];
#pragma unroll
      for (int u = 0; u < UN; ++u) {
        const int k = (c + u) * F::K + quad * F::PER;
        xf[u] = ld_frag<T, WHOLE>(xr, k, a.D);
#pragma unroll
        for (int i = 0; i < 4; ++i) wf[u][i] = ld_frag<T, WHOLE>(wr[i], k, a.D);
      }
#pragma unroll
      for (int u = 0; u < UN; ++u)
#pragma unroll
        for (int i = 0; i < 4; ++i) acc[i] = mma(wf[u][i], xf[u], acc[i]);
    };
    int c = wave * 4;
    for (; c + 4 <= steps; c += 4 * RW) run(c, std::integral_constant<int, 4>());
    for (; c < steps; ++c) run(c, std::integral_constant<int, 1>());
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
      for (int r = 0; r < 4; ++r) part[(wave * RT + col) * 65 + i * 16 + quad * 4 + r] = acc[i][r];
    __syncthreads();
    for (int i = threadIdx.x; i < RT * 64; i += 64 * RW) {
      const int t = i >> 6, e = e0 + (i & 63);
      if (e < Z) {
        float z = 0.f;
#pragma unroll
        for (int v = 0; v < RW; ++v) z += part[(v * RT + t) * 65 + (i & 63)];
        const float s = a.softmax && e < a.E ? z : 1.f / (1.f + expf(-z));
        if (e < a.E) {
          score[t * a.E + e] = s;
          choice[t * a.E + e] = correction ? s + ld(correction + e) : s;
        } else open[t] = s;
      }
    }
    __syncthreads();
  }
  const int size = a.E / a.groups;
  const int t = threadIdx.x >> 4, l = threadIdx.x & 15;
  if (t < RT) {  // rows of LDS are the sixteen lanes' own
    float* ch = choice + t * a.E;
    if (a.keep < a.groups) {
      // lane l (and l + 16, ..) scores group l by its two best
      float* gs = part + t * a.groups;
      for (int g = l; g < a.groups; g += 16) {
        float b1 = -INFINITY, b2 = -INFINITY;
#pragma unroll 4
        for (int i = 0; i < size; ++i) {
          const float v = ch[g * size + i];
          b2 = fmaxf(b2, fminf(v, b1));
          b1 = fmaxf(b1, v);
        }
        gs[g] = size > 1 ? b1 + b2 : b1;
      }
      __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
      for (int g = l; g < a.groups; g += 16) {
        const float mine = gs[g];
        int better = 0;
        for (int o = 0; o < a.groups; ++o) better += gs[o] > mine || (gs[o] == mine && o < g);
        if (better >= a.keep)
          for (int i = 0; i < size; ++i) ch[g * size + i] = -INFINITY;
      }
      __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
    }
    float v[J];
#pragma unroll
    for (int j = 0; j < J; ++j) v[j] = l + j * 16 < a.E ? ch[l + j * 16] : -INFINITY;
    const bool valid = t0 + t < a.T;
    float mine = 0.f;  // score of the choice that lane l weighs
    for (int k = 0; k < a.pick; ++k) {
      float best = v[0];
#pragma unroll
      for (int j = 1; j < J; ++j) best = fmaxf(best, v[j]);
      best = row_max(best);
      int at = INT_MAX;
#pragma unroll
      for (int j = J - 1; j >= 0; --j)
        if (v[j] == best) at = l + j * 16;
      at = min(row_min(at), a.E - 1);  // the lowest of equals
#pragma unroll
      for (int j = 0; j < J; ++j)
        if (at == l + j * 16) v[j] = -INFINITY;
      if (l == k) mine = score[t * a.E + at];
      if (l == 0) {
        chosen[t * a.top + k] = valid ? at : -1;
        if (valid) idx[(size_t)(t0 + t) * a.top + k] = at;
      }
    }
    if (a.softmax) {
      const float e = l < a.pick ? expf(mine - row_max(l < a.pick ? mine : -INFINITY)) : 0.f;
      mine = e / row_sum(e);
    }
    if (valid && l < a.pick) weight[(size_t)(t0 + t) * a.top + l] = mine * a.scale;
    for (int k = a.pick + l; k < a.top; k += 16) {
      const int e = a.E + k - a.pick;
      chosen[t * a.top + k] = valid ? e : -1;
      if (valid) {
        idx[(size_t)(t0 + t) * a.top + k] = e;
        weight[(size_t)(t0 + t) * a.top + k] = a.gate ? open[t] : 1.f;
      }
    }
  }
  __syncthreads();
  // place among the block's pairs of the same expert, and the block's counts;
  // chosen holds RT * top entries, a multiple of four
  const int4* four = (const int4*)chosen;
  const int pairs = (min(RT, a.T - t0) * a.top + 3) >> 2;  // fours of them
  for (int e = threadIdx.x; e < a.all; e += 64 * RW) {
    int n = 0;
    int* dst = rank + (size_t)t0 * a.top;
    for (int o = 0; o < pairs; ++o) {
      const int4 c = four[o];
      if (c.x == e) dst[o * 4] = n++;
      if (c.y == e) dst[o * 4 + 1] = n++;
      if (c.z == e) dst[o * 4 + 2] = n++;
      if (c.w == e) dst[o * 4 + 3] = n++;
    }
    counts[(size_t)e * a.nblk + blockIdx.x] = n;
  }
}

// counts [E][nblk] -> exclusive sums along nblk, in place, and the totals [E]
__global__ __launch_bounds__(256) void count_scan_kernel(int* __restrict__ counts, int* __restrict__ total, int nblk) {
  __shared__ int sums[256];
  int* row = counts + (size_t)blockIdx.x * nblk;
  const int per = (nblk + 255) / 256, lo = threadIdx.x * per, hi = min(lo + per, nblk);
  int n = 0;
  for (int i = lo; i < hi; ++i) n += row[i];
  sums[threadIdx.x] = n;
  __syncthreads();
  for (int d = 1; d < 256; d <<= 1) {
    const int o = threadIdx.x >= d ? sums[threadIdx.x - d] : 0;
    __syncthreads();
    sums[threadIdx.x] += o;
    __syncthreads();
  }
  int at = sums[threadIdx.x] - n;
  for (int i = lo; i < hi; ++i) {
    const int c = row[i];
    row[i] = at;
    at += c;
  }
  if (threadIdx.x == 255) total[blockIdx.x] = sums[255];
}

// Rows of all pairs: row[pair], token[row] and, by_row given, the pair's weight;
// first row of every expert [E + 1]; tiles (expert, first row), expert -1 past
// the last.
__global__ __launch_bounds__(256) void place_kernel(
    const int* __restrict__ idx, const int* __restrict__ rank, const int* __restrict__ before,
    const int* __restrict__ total, const float* __restrict__ weight, int* __restrict__ row, int* __restrict__ token,
    float* __restrict__ by_row, int* __restrict__ first, int2* __restrict__ tiles, int max_tiles, RouteArgs a) {
  __shared__ int at[MAX_EXPERTS], cnt[MAX_EXPERTS], tile_at[MAX_EXPERTS], ends[2];
  // a single block of the router needs no scan: its counts are the totals
  for (int e = threadIdx.x; e < a.all; e += 256) cnt[e] = a.nblk == 1 ? before[e] : total[e];
  __syncthreads();
  if (threadIdx.x < 64) {  // one wave scans, E/64 each
    const int per = (a.all + 63) / 64, lo = threadIdx.x * per, hi = min(lo + per, a.all);
    int n = 0, m = 0;
    for (int e = lo; e < hi; ++e) { n += cnt[e]; m += (cnt[e] + a.tile - 1) / a.tile; }
    int sn = n, sm = m;
#pragma unroll
    for (int d = 1; d < 64; d <<= 1) {
      const int on = __shfl_up(sn, d), om = __shfl_up(sm, d);
      if (threadIdx.x >= d) { sn += on; sm += om; }
    }
    if (threadIdx.x == 63) { ends[0] = sn; ends[1] = sm; }
    sn -= n;
    sm -= m;
    for (int e = lo; e < hi; ++e) {
      at[e] = sn;
      tile_at[e] = sm;
      sn += cnt[e];
      sm += (cnt[e] + a.tile - 1) / a.tile;
    }
  }
  __syncthreads();
  const int pair = blockIdx.x * 256 + threadIdx.x;
  if (pair < a.T * a.top) {
    const int e = idx[pair], t = pair / a.top;
    const int r = at[e] + (a.nblk == 1 ? 0 : before[(size_t)e * a.nblk + t / RT]) + rank[pair];
    row[pair] = r;
    token[r] = t;
    if (by_row) by_row[r] = weight[pair];
  }
  if (blockIdx.x) return;
  for (int e = threadIdx.x; e < a.all; e += 256) {
    first[e] = at[e];
    for (int i = 0; i * a.tile < cnt[e]; ++i) tiles[tile_at[e] + i] = make_int2(e, at[e] + i * a.tile);
  }
  for (int i = ends[1] + threadIdx.x; i < max_tiles; i += 256) tiles[i] = make_int2(-1, 0);
  if (threadIdx.x == 0) first[a.all] = ends[0];
}

// ---------------------------------------------------------------------------
// grouped products
// ---------------------------------------------------------------------------

struct Act { float alpha, limit, plus; };
// min(g, limit) sigmoid(alpha min(g, limit)) (clamp(u, -limit, limit) + plus)
DEVINL float gated(float g, float u, const Act& a) {
  g = fminf(g, a.limit);
  u = fminf(fmaxf(u, -a.limit), a.limit);
  return g * sigmoidf(a.alpha * g) * (u + a.plus);
}

// What a product is: of a pair's own row; of its token with gate and up weights
// and the gated activation; of its token with one set of weights and the square
// of what is positive.
enum Product { PLAIN, GATED, RELU2 };

struct GroupArgs {
  int K, kp, F, E;  // valid and stored length of a weight row, output features, experts
  int xs, ys;       // row strides of input and output
};

// A product's rows times what scales them, through its activation
template <int KIND>
DEVINL float activated(float by, float g, float u, const Act& a) {
  if (KIND == GATED) return gated(by * g, by * u, a);
  g = by * g;
  if (KIND == RELU2) g = fmaxf(g, 0.f) * g;
  return g;
}

// Few tokens per expert: a block owns 16 output features of one expert; its
// four waves split k and walk the expert's rows up to 64 (GATED: 32) at a time. GATED:
// weights [E][2][F][kp]; else [E][F][kp]. Input rows are gathered by token but
// for PLAIN. by_row: what the rows of the product are scaled with.
template <typename T, int KIND, bool WHOLE>
__global__ __launch_bounds__(256) void expert_stream_kernel(
    const T* __restrict__ x, const T* __restrict__ w, const int* __restrict__ first, const int* __restrict__ token,
    const float* __restrict__ by_row, T* __restrict__ y, GroupArgs a, Act act) {
  typedef Frag<T> F;
  constexpr int NW = KIND == GATED ? 2 : 1, MOST = 4 / NW;
  __shared__ float part[4][NW][MOST * 16][17];
  // the last experts are the ones that every token uses: the longest come first
  const int e = gridDim.y - 1 - blockIdx.y, f0 = blockIdx.x * 16;
  const int lo = first[e], hi = first[e + 1];
  if (lo == hi) return;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, col = lane & 15, quad = lane >> 4;
  const T* wr[NW];
#pragma unroll
  for (int i = 0; i < NW; ++i) wr[i] = w + (((size_t)e * NW + i) * a.F + f0 + col) * a.kp + quad * F::PER;
  const int steps = (a.K + F::K - 1) / F::K;
  auto round = [&](int r0, auto tiles) {  // 16 * MT rows
    constexpr int MT = decltype(tiles)::value, UN = MT == 4 ? 4 : 8 / NW;
    floatx4 acc[NW][MT];
    const T* xr[MT];
#pragma unroll
    for (int m = 0; m < MT; ++m) {
      const int r = min(r0 + m * 16 + col, hi - 1);
      xr[m] = x + (size_t)(KIND == PLAIN ? r : token[r]) * a.xs;
#pragma unroll
      for (int i = 0; i < NW; ++i) acc[i][m] = (floatx4)(0.f);
    }
    auto run = [&](int c, auto count) {  // `count` steps from c on, loads first
      constexpr int N = decltype(count)::value;
      typename F::V wf[N][NW], xf[N][MT];
#pragma unroll
      for (int u = 0; u < N; ++u) {
#pragma unroll
        for (int i = 0; i < NW; ++i) wf[u][i] = *(const typename F::V*)(wr[i] + (size_t)(c + u) * F::K);
#pragma unroll
        for (int m = 0; m < MT; ++m) xf[u][m] = ld_frag<T, WHOLE>(xr[m], (c + u) * F::K + quad * F::PER, a.K);
      }
#pragma unroll
      for (int u = 0; u < N; ++u)
#pragma unroll
        for (int m = 0; m < MT; ++m)
#pragma unroll
          for (int i = 0; i < NW; ++i) acc[i][m] = mma(wf[u][i], xf[u][m], acc[i][m]);
    };
    int c = wave * UN;
    for (; c + UN <= steps; c += 4 * UN) run(c, std::integral_constant<int, UN>());
    for (; c < steps; ++c) run(c, std::integral_constant<int, 1>());
#pragma unroll
    for (int i = 0; i < NW; ++i)
#pragma unroll
      for (int m = 0; m < MT; ++m)
#pragma unroll
        for (int r = 0; r < 4; ++r) part[wave][i][m * 16 + col][quad * 4 + r] = acc[i][m][r];
    __syncthreads();
    const int n = min(16 * MT, hi - r0);
    for (int i = threadIdx.x; i < n * 16; i += 256) {
      const int t = i >> 4, f = i & 15;
      float v[NW];
#pragma unroll
      for (int j = 0; j < NW; ++j)
        v[j] = part[0][j][t][f] + part[1][j][t][f] + part[2][j][t][f] + part[3][j][t][f];
      const float by = KIND != PLAIN && by_row ? by_row[r0 + t] : 1.f;
      st(y + (size_t)(r0 + t) * a.ys + f0 + f, activated<KIND>(by, v[0], v[NW - 1], act));
    }
    __syncthreads();
  };
  int r0 = lo;
  for (; hi - r0 > 32; r0 += MOST * 16) round(r0, std::integral_constant<int, MOST>());
  if (hi - r0 > 16) round(r0, std::integral_constant<int, 2>());
  else if (hi > r0) round(r0, std::integral_constant<int, 1>());
}

// Many tokens per expert (bf16): TOK tokens x 256 weight rows (GATED: 128 gate
// and the same 128 up) per block, a wave 64 x 128 of it, k in steps of 64
// through 2 (TOK 256) or 3 LDS buffers. LDS rows hold 8 pieces of 16 bytes,
// piece p of row r at place p ^ (r & 7): loads go straight to LDS lane by lane,
// so the permutation sits in the global address, and fragment reads spread
// over the banks.
constexpr int TILE_W = 256;  // weight rows

template <int TOK> struct TileShape {
  static constexpr int WAVES = TOK / 32, BUFS = TOK == 256 ? 2 : 3, BUF = (TILE_W + TOK) * 64;  // elements of a buffer
};

template <int KIND, int TOK>
__global__ __launch_bounds__(TOK * 2) void expert_tile_kernel(
    const bf16_t* __restrict__ x, const bf16_t* __restrict__ w, const int* __restrict__ first,
    const int* __restrict__ token, const int2* __restrict__ tiles, const float* __restrict__ by_row,
    bf16_t* __restrict__ y, int max_tiles, int group, GroupArgs a, Act act) {
  typedef TileShape<TOK> Sh;
  constexpr bool TWO = KIND == GATED;  // weight rows are gate and up
  constexpr int WL = TILE_W / Sh::WAVES / 8, XL = 4, LOADS = WL + XL;  // loads of a stage and wave
  extern __shared__ __attribute__((aligned(16))) bf16_t buf[];  // [BUFS][weights [256][64], tokens [TOK][64]]
  // blocks go round the eight dies: give a die `group` neighbouring tiles and
  // all their features, so that its L2 serves both operands
  const int nf = (a.F + (TWO ? 127 : 255)) / (TWO ? 128 : 256);
  const int local = blockIdx.x >> 3, per = group * nf;
  const int m = (local / per * 8 + (blockIdx.x & 7)) * group + local % group, fb = local % per / group;
  if (m >= max_tiles) return;
  const int2 tile = tiles[m];
  if (tile.x < 0) return;
  const int hi = first[tile.x + 1], r0 = tile.y;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int lane = threadIdx.x & 63, col = lane & 15, quad = lane >> 4;
  const int wf = wave & 1, wt = wave >> 1;  // which 128 weight rows, which 64 tokens
  const int f0 = fb * (TWO ? 128 : 256);
  // each wave stages its share of the weight rows and 32 tokens, 8 rows a load
  const bf16_t *wsrc[WL], *xsrc[XL];
  const int piece = ((lane & 7) ^ (lane >> 3)) * 8;
#pragma unroll
  for (int i = 0; i < WL; ++i) {
    const int r = (wave * WL + i) * 8 + (lane >> 3);
    // GATED rows: [64 gate, the same 64 up] for either half of the features
    const int f = TWO ? f0 + (r >> 7) * 64 + (r & 63) : f0 + r;
    const int part = TWO ? (r >> 6) & 1 : 0;
    wsrc[i] = w + (((size_t)tile.x * (TWO ? 2 : 1) + part) * a.F + min(f, a.F - 1)) * a.kp + piece;
  }
#pragma unroll
  for (int i = 0; i < XL; ++i) {
    const int t = min(r0 + wave * 32 + i * 8 + (lane >> 3), hi - 1);
    xsrc[i] = x + (size_t)(KIND == PLAIN ? t : token[t]) * a.xs;
  }
  auto stage = [&](int s) {
    const int k = s * 64;
    bf16_t* dst = buf + (s % Sh::BUFS) * Sh::BUF;
#pragma unroll
    for (int i = 0; i < WL; ++i)
      __builtin_amdgcn_global_load_lds((const __attribute__((address_space(1))) void*)(wsrc[i] + k),
                                       (__attribute__((address_space(3))) void*)(dst + (wave * WL + i) * 512), 16, 0, 0);
    // past the end of a row the weights are zero; any number of the row will do
    const int kx = k + piece < a.K ? k + piece : 0;
#pragma unroll
    for (int i = 0; i < XL; ++i)
      __builtin_amdgcn_global_load_lds((const __attribute__((address_space(1))) void*)(xsrc[i] + kx),
                                       (__attribute__((address_space(3))) void*)(dst + (TILE_W + wave * 32 + i * 8) * 64), 16, 0, 0);
  };
  floatx4 acc[8][4];
#pragma unroll
  for (int i = 0; i < 8; ++i)
#pragma unroll
    for (int j = 0; j < 4; ++j) acc[i][j] = (floatx4)(0.f);
  const int steps = (a.K + 63) / 64;
  stage(0);
  if (Sh::BUFS == 3 && steps > 1) stage(1);
  // a lane's fragments, as LDS byte addresses within a buffer
  const unsigned wl = (unsigned)(size_t)(__attribute__((address_space(3))) bf16_t*)(buf + (wf * 128 + col) * 64);
  const unsigned xl = (unsigned)(size_t)(__attribute__((address_space(3))) bf16_t*)(buf + (TILE_W + wt * 64 + col) * 64);
  const unsigned place[2] = {(unsigned)((quad ^ (col & 7)) * 16), (unsigned)(((4 + quad) ^ (col & 7)) * 16)};
  for (int s = 0; s < steps; ++s) {
    // this step is in LDS (of three buffers, the next may still be on its
    // way); the buffer of the one before is free
    if (Sh::BUFS == 3 && s + 1 < steps) asm volatile("s_waitcnt vmcnt(%0)\n\ts_barrier" ::"i"(LOADS) : "memory");
    else asm volatile("s_waitcnt vmcnt(0)\n\ts_barrier" ::: "memory");
    const unsigned at = (unsigned)(s % Sh::BUFS) * (Sh::BUF * 2);
    // reads by hand: the compiler would make them wait for every pending load to LDS
    constexpr int SETS = Sh::BUFS == 3 ? 2 : 1;  // halves of the step in registers at a time
    bf16x8 wv[SETS][8], xv[SETS][4];
    auto read = [&](int kk, bf16x8* w8, bf16x8* x4) {
      const unsigned wa = wl + at + place[kk], xa = xl + at + place[kk];
#define READ(D, A, I) asm volatile("ds_read_b128 %0, %1 offset:%2" : "=v"(D) : "v"(A), "i"((I) * 2048))
      READ(x4[0], xa, 0); READ(x4[1], xa, 1); READ(x4[2], xa, 2); READ(x4[3], xa, 3);
      READ(w8[0], wa, 0); READ(w8[1], wa, 1); READ(w8[2], wa, 2); READ(w8[3], wa, 3);
      READ(w8[4], wa, 4); READ(w8[5], wa, 5); READ(w8[6], wa, 6); READ(w8[7], wa, 7);
#undef READ
    };
#pragma unroll
    for (int kk = 0; kk < SETS; ++kk) read(kk, wv[kk], xv[kk]);
    if (s + Sh::BUFS - 1 < steps) stage(s + Sh::BUFS - 1);
#pragma unroll
    for (int kk = 0; kk < 2; ++kk) {
      bf16x8 *w8 = wv[kk % SETS], *x4 = xv[kk % SETS];
      if (SETS == 1 && kk == 1) read(1, w8, x4);
      // 12 reads of the second half may be pending while the first is used
#define TIE(D) "+v"(D)
#define WAIT(N)                                                                                                       \
  asm volatile("s_waitcnt lgkmcnt(" #N ")" : TIE(x4[0]), TIE(x4[1]), TIE(x4[2]), TIE(x4[3]), TIE(w8[0]), TIE(w8[1]), \
               TIE(w8[2]), TIE(w8[3]), TIE(w8[4]), TIE(w8[5]), TIE(w8[6]), TIE(w8[7]))
      if (SETS == 2 && kk == 0) WAIT(12);
      else WAIT(0);
#undef WAIT
#undef TIE
#pragma unroll
      for (int i = 0; i < 8; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j) acc[i][j] = mma(w8[i], x4[j], acc[i][j]);
    }
  }
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    const int t = r0 + wt * 64 + j * 16 + col;
    if (t >= hi) continue;
    bf16_t* dst = y + (size_t)t * a.ys;
    const float by = KIND != PLAIN && by_row ? by_row[t] : 1.f;
    constexpr int N = TWO ? 4 : 8;
#pragma unroll
    for (int i = 0; i < N; ++i) {
      const int f = f0 + wf * 16 * N + i * 16 + quad * 4;
      float v[4];
#pragma unroll
      for (int r = 0; r < 4; ++r) v[r] = activated<KIND>(by, acc[i][j][r], acc[(i + 4) & 7][j][r], act);
      if (f < a.F) st4(dst + f, v);
    }
  }
}

// ---------------------------------------------------------------------------
// residual sum and norm
// ---------------------------------------------------------------------------

// x += mult * y (top 0) or mult * sum_j weight_j y[row_j]; h = norm(x; w_next).
// One block per token; the row stays in registers.
template <typename T, int V, int NC>
__global__ __launch_bounds__(256) void add_norm_kernel(
    const T* __restrict__ y, const int* __restrict__ rows, const float* __restrict__ weight, int top, int ys,
    float* __restrict__ x, const T* __restrict__ w_next, T* __restrict__ h, int D, float mult, float eps) {
  const size_t off = (size_t)blockIdx.x * D;
  __shared__ float red[4];
  float xv[NC * V], acc = 0.f;
#pragma unroll
  for (int c = 0; c < NC; ++c) {
    const int i = (c * 256 + threadIdx.x) * V;
    float sum[V];
#pragma unroll
    for (int j = 0; j < V; ++j) xv[c * V + j] = sum[j] = 0.f;
    if (i < D) {
      ldv<V>(x + off + i, xv + c * V);
      if (top == 0) ldv<V>(y + (size_t)blockIdx.x * ys + i, sum);
      for (int k = 0; k < top; ++k) {
        const float wk = weight ? weight[(size_t)blockIdx.x * top + k] : 1.f;
        float v[V];
        ldv<V>(y + (size_t)rows[(size_t)blockIdx.x * top + k] * ys + i, v);
#pragma unroll
        for (int j = 0; j < V; ++j) sum[j] += wk * v[j];
      }
#pragma unroll
      for (int j = 0; j < V; ++j) {
        xv[c * V + j] += mult * sum[j];
        acc += xv[c * V + j] * xv[c * V + j];
      }
      stv<V>(x + off + i, xv + c * V);
    }
  }
  if (!w_next) return;
  const float inv = 1.f / sqrtf(block_sum(acc, red) / (float)D + eps);
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

// ===========================================================================
// host side
// ===========================================================================

// x [.., D] -> (weights [T, top] fp32, row of every pair [T, top], token of
// every row, first row of every expert [E + 1], tiles [max, 2], rows of a tile).
// `shared` experts follow the routed ones in every token's list (top counts
// them then); their weight is the sigmoid of one more row of w (gate) or one.
// on_input: the weights by row [T * top].
std::tuple<Tensor, Tensor, Tensor, Tensor, Tensor, int64_t> route(Tensor x, Tensor w, OptT correction, int64_t pick,
                                                                  int64_t groups, int64_t keep, double scale,
                                                                  bool softmax, int64_t shared, bool gate,
                                                                  bool on_input) {
  const auto dt = io_type(x);
  check_io(w, dt);
  gate = gate && shared > 0;
  const int D = x.size(-1), T_ = x.numel() / D, E = w.size(0) - gate;
  if (correction) { check_io(*correction, dt); CHK(correction->numel() == E); }
  CHK(w.dim() == 2 && w.size(1) == D && T_ > 0 && shared >= 0);
  const int64_t top = pick + shared, all = E + shared;
  TORCH_CHECK(E >= 1 && all <= MAX_EXPERTS && pick >= 1 && pick <= MAX_PICK && pick <= E, "routing to ", pick, " of ", E,
              " experts and ", shared, " shared ones");
  TORCH_CHECK(groups >= 1 && E % groups == 0 && keep >= 1 && keep <= groups && pick <= keep * (E / groups),
              "routing to ", pick, " experts of ", keep, " of ", groups, " groups of ", E, " experts");
  CHK((int64_t)T_ * top < INT_MAX);
  const int nblk = (T_ + RT - 1) / RT, pairs = T_ * (int)top;
  const int tile = pairs >= 320 * all ? 256 : 128, max_tiles = pairs / tile + std::min(pairs, (int)all);
  const auto ints = x.options().dtype(torch::kInt32);
  auto weight = f32(x, {T_, top});
  Tensor by_row;
  if (on_input) by_row = f32(x, {pairs});
  auto idx = torch::empty({T_, top}, ints), rank = torch::empty({T_, top}, ints), row = torch::empty({T_, top}, ints);
  auto counts = torch::empty({all, nblk}, ints), total = torch::empty({all}, ints), first = torch::empty({all + 1}, ints);
  auto token = torch::empty({pairs}, ints), tiles = torch::empty({max_tiles, 2}, ints);
  const RouteArgs a{T_, D, E, (int)top, (int)groups, (int)keep, nblk, tile, (float)scale, (int)pick, (int)all, softmax, gate};
  const hipStream_t stream = cur_stream();
  CHK(groups <= 4 * 65);
  BY_TYPE(dt, {
    const T* cp = correction ? P<T>(*correction) : nullptr;
    auto run = [&](auto kernel, int waves) {
      static const hipError_t err = hipFuncSetAttribute((const void*)kernel, hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
      TORCH_CHECK(err == hipSuccess, "no LDS for the router");
      const size_t lds = (2 * RT * E + waves * RT * 65) * sizeof(float) + RT * (top + 1) * sizeof(int);  // parts of 16 bytes
      hipLaunchKernelGGL(kernel, dim3(nblk), dim3(64 * waves), lds, stream, P<T>(x), P<T>(w), cp,
                         idx.data_ptr<int>(), M<float>(weight), rank.data_ptr<int>(), counts.data_ptr<int>(), a);
    };
    // few tokens: more waves on each
    const bool few = nblk <= 256;
    if (D % Frag<T>::K) run(route_kernel<T, false, MAX_EXPERTS / 16, 4>, 4);
    else if (E <= 64) { if (few) run(route_kernel<T, true, 4, 16>, 16); else run(route_kernel<T, true, 4, 4>, 4); }
    else if (E <= 256) { if (few) run(route_kernel<T, true, 16, 16>, 16); else run(route_kernel<T, true, 16, 4>, 4); }
    else run(route_kernel<T, true, MAX_EXPERTS / 16, 4>, 4);
  });
  if (nblk > 1)
    hipLaunchKernelGGL(count_scan_kernel, dim3(all), dim3(256), 0, stream, counts.data_ptr<int>(), total.data_ptr<int>(), nblk);
  hipLaunchKernelGGL(place_kernel, dim3((pairs + 255) / 256), dim3(256), 0, stream, idx.data_ptr<int>(),
                     rank.data_ptr<int>(), counts.data_ptr<int>(), total.data_ptr<int>(), P<float>(weight),
                     row.data_ptr<int>(), token.data_ptr<int>(), on_input ? M<float>(by_row) : nullptr,
                     first.data_ptr<int>(), (int2*)tiles.data_ptr<int>(), max_tiles, a);
  return {on_input ? by_row : weight, row, token, first, tiles, tile};
}

// One grouped product over all pairs: GATED (x by token, weights [E,2,F,kp]),
// RELU2 (x by token, weights [E,F,kp]) or PLAIN (x by row, weights [E,F,kp]); kp:
// row length padded with zeros. by_row [pairs]: scales of the product's rows.
Tensor expert_product(Tensor x, Tensor w, Tensor token, Tensor first, Tensor tiles, int64_t tile, int64_t kind,
                      double alpha, double limit, double plus, OptT by_row) {
  const auto dt = io_type(x);
  check_io(w, dt);
  CHK(kind == PLAIN || kind == GATED || kind == RELU2);
  const bool gated_ = kind == GATED;
  CHK(w.dim() == (gated_ ? 4 : 3) && x.dim() == 2);
  for (const Tensor& t : {token, first, tiles}) check_io(t, torch::kInt32);
  const int E = w.size(0), F_ = w.size(-2), kp = w.size(-1), K = x.size(1), pairs = token.numel();
  CHK((!gated_ || w.size(1) == 2) && first.numel() == E + 1 && K <= kp && kp % 64 == 0 && F_ % 16 == 0 && kp - K < 64);
  CHK(kind != PLAIN || x.size(0) == pairs);
  if (by_row) { check_io(*by_row, torch::kFloat32); CHK(kind != PLAIN && by_row->numel() == pairs); }
  const float* bp = by_row ? P<float>(*by_row) : nullptr;
  auto y = torch::empty({pairs, F_}, x.options());
  const GroupArgs a{K, kp, F_, E, K, F_};
  const Act act{(float)alpha, (float)limit, (float)plus};
  const hipStream_t stream = cur_stream();
  const int *fp = first.data_ptr<int>(), *tp = token.data_ptr<int>();
  // on average more than 24 rows per expert: weights are worth tiling
  if (dt == torch::kBFloat16 && K % 8 == 0 && pairs > 24 * E) {
    const int width = gated_ ? TILE_W / 2 : TILE_W;
    const int max_tiles = tiles.size(0), group = std::min(8, std::max(1, max_tiles / 64)), nf = (F_ + width - 1) / width;
    const dim3 grid((max_tiles + 8 * group - 1) / (8 * group) * 8 * group * nf);
    const int2* tl = (const int2*)tiles.data_ptr<int>();
    CHK(tile == 128 || tile == 256);
    auto run = [&](auto kernel, int threads, int lds) {
      static const hipError_t err = hipFuncSetAttribute((const void*)kernel, hipFuncAttributeMaxDynamicSharedMemorySize, lds);
      TORCH_CHECK(err == hipSuccess, "no LDS for expert tiles");
      hipLaunchKernelGGL(kernel, grid, dim3(threads), lds, stream, P<bf16_t>(x), P<bf16_t>(w), fp, tp, tl, bp,
                         M<bf16_t>(y), max_tiles, group, a, act);
    };
#define TILES(KIND, TOK) \
  run(expert_tile_kernel<KIND, TOK>, TOK * 2, TileShape<TOK>::BUFS * TileShape<TOK>::BUF * (int)sizeof(bf16_t))
#define TILES_OF(KIND) if (tile == 256) TILES(KIND, 256); else TILES(KIND, 128)
    if (kind == GATED) { TILES_OF(GATED); }
    else if (kind == RELU2) { TILES_OF(RELU2); }
    else { TILES_OF(PLAIN); }
#undef TILES_OF
#undef TILES
    return y;
  }
  const dim3 grid(F_ / 16, E);
#define STREAM(KIND, WHOLE)                                                                                     \
  hipLaunchKernelGGL((expert_stream_kernel<T, KIND, WHOLE>), grid, dim3(256), 0, stream, P<T>(x), P<T>(w), fp,     \
                     tp, bp, M<T>(y), a, act)
#define STREAM_OF(KIND) if (K % Frag<T>::K == 0) STREAM(KIND, true); else STREAM(KIND, false);
  BY_TYPE(dt, {
    if (kind == GATED) { STREAM_OF(GATED) }
    else if (kind == RELU2) { STREAM_OF(RELU2) }
    else { STREAM_OF(PLAIN) }
  });
#undef STREAM_OF
#undef STREAM
  return y;
}

// x += mult * y, or mult * the weighted rows of y; returns the stream's norm
OptT add_norm(Tensor y, OptT rows, OptT weight, Tensor x, OptT w_next, double mult, double eps) {
  const auto dt = io_type(y);
  check_io(x, torch::kFloat32);
  const int D = x.size(-1), n = x.numel() / D, ys = y.size(-1);
  int top = 0;
  if (rows) {
    check_io(*rows, torch::kInt32);
    if (weight) { check_io(*weight, torch::kFloat32); CHK(weight->numel() == rows->numel()); }
    top = rows->size(-1);
    CHK(rows->numel() == (int64_t)n * top && y.numel() == (int64_t)n * top * ys && ys >= D);
  } else {
    CHK(y.numel() == x.numel() && ys == D);
  }
  OptT h;
  if (w_next) { check_io(*w_next, dt); CHK(w_next->numel() == D); h = torch::empty(x.sizes(), x.options().dtype(dt)); }
  if (n == 0) return h;
  const int* rp = rows ? rows->data_ptr<int>() : nullptr;
  const float* wp = weight ? weight->data_ptr<float>() : nullptr;
#define NORM(V, NC)                                                                                            \
  if (nc <= NC) {                                                                                              \
    hipLaunchKernelGGL((add_norm_kernel<T, V, NC>), dim3(n), dim3(256), 0, cur_stream(), P<T>(y), rp, wp, top, ys, \
                       M<float>(x), wn, hp, D, (float)mult, (float)eps);                                       \
    return h;                                                                                                  \
  }
  BY_TYPE(dt, {
    const T* wn = w_next ? P<T>(*w_next) : nullptr;
    T* hp = h ? M<T>(*h) : nullptr;
    if (D % 4 == 0 && ys % 4 == 0) {
      const int nc = (D + 1023) / 1024;
      NORM(4, 1) NORM(4, 2) NORM(4, 4) NORM(4, 8) NORM(4, 16)
    } else {
      const int nc = (D + 255) / 256;
      NORM(1, 1) NORM(1, 4) NORM(1, 16)
    }
  });
#undef NORM
  TORCH_CHECK(false, "row of ", D, " elements is too long");
}

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.def("route", &route, "router: sigmoid scores or a softmax over the chosen, group-limited top-k, shared experts; rows of all pairs",
        py::arg("x"), py::arg("w"), py::arg("correction"), py::arg("top"), py::arg("groups"), py::arg("keep"),
        py::arg("scale"), py::arg("softmax") = false, py::arg("shared") = 0, py::arg("gate") = true,
        py::arg("on_input") = false);
  m.def("expert_product", &expert_product, "grouped product of all (token, expert) pairs, with an activation or plain",
        py::arg("x"), py::arg("w"), py::arg("token"), py::arg("first"), py::arg("tiles"), py::arg("tile"), py::arg("kind"),
        py::arg("alpha") = 0.0, py::arg("limit") = 0.0, py::arg("plus") = 0.0, py::arg("by_row") = py::none());
  m.attr("PLAIN") = (int)PLAIN;
  m.attr("GATED") = (int)GATED;
  m.attr("RELU2") = (int)RELU2;
  m.def("add_norm", &add_norm, "stream += mult * (output or weighted expert rows); norm of the stream");
}
