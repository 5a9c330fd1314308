// CDNA4 (gfx950) kernels of matrix memories with exponential gates (the mLSTM
// of xLSTM). Per head, with logs i and f of the input and forget gate,
//   m_t = max(f_t + m_(t-1), i_t)                       m starts at 0
//   S_t = e^{f_t + m_(t-1) - m_t} S_(t-1) + e^{i_t - m_t} k_t v_t^T
//   o_t = S_t^T q_t / (max(|n_t q_t|, e^{-m_t}) + 1e-6)  n: S with v = 1
// and o's RMS norm per head, a weight and a sigmoid gate. Gates, state, decays
// and norms are fp32; q, k, v are bf16 or fp32.
//
// Prompts: gates_kernel makes the running maximum of a whole row, so that
// chunks of tokens know theirs; memory_kernel walks the chunks. With F_t the log
// forget gates of a chunk summed up to t, u_t = F_t - m_t and r_s = i_s - F_s:
//   O_t = e^{u_t + m} q_t S + sum_{s<=t} e^{u_t + r_s} (q_t k_s) v_s
//   S'  = e^{u_C + m} S + sum_s e^{u_C + r_s} k_s v_s^T
// (m: the maximum before the chunk, C: its last token). No exponent is positive.
// Decays scale whole tokens, so q, k and v enter the products as they are; what
// is fp32 (S, decayed v, scores) enters bf16 products as a sum of two bf16
// parts, which keeps 16 bits of mantissa. i, f, m, u and r are kept as logarithms
// to base 2.
//
// Rows of a step address state by slot (struct Step): slot -1 is a parked row,
// which reads and writes no state and yields zeros. A row at position 0
// ignores what its slot holds.

#include "common.h"

struct MemArgs {
  int S, H, N, K;                            // tokens, heads, widths of input and output
  int q_at, k_at, v_at, g_at, i_at, f_at, out_at;
  int dim, vdim, dp;                         // dp: key channels of a state row
  int P;                                     // tokens of a row in whole chunks
  int seg, nseg;                             // chunks of a segment, segments
  float cap, eps, scale, out_scale;
};

constexpr int C = 32;  // tokens of a chunk

// log gates of a token: cap tanh((z + b) / cap), of the forget gate through logsigmoid
constexpr float LOG2E = 1.4426950408889634f;
DEVINL float capped(float z, float bias, float cap) { return cap * tanhf((z + bias) / cap); }
DEVINL float log_input(float z, float bias, float cap) { return LOG2E * capped(z, bias, cap); }
DEVINL float log_forget(float z, float bias, float cap) {
  const float x = capped(z, bias, cap);
  return LOG2E * (fminf(x, 0.f) - log1pf(expf(-fabsf(x))));
}
DEVINL float pow2(float x) { return __builtin_amdgcn_exp2f(x); }

// One block per (head, row): u, r [B][H][P] and m [B][H][P + 1], m[0] that before
// the row. A thread has `per` tokens (a power of two, so that chunks begin at
// threads or threads at chunks), PER of them in registers; PER 0: any number, kept
// in u and r between the two walks.
template <typename T, int PER>
__global__ __launch_bounds__(256) void gates_kernel(
    const T* __restrict__ proj, const T* __restrict__ bias, float* __restrict__ state_m, float* u, float* r,
    float* __restrict__ m, int per, MemArgs a, Step step) {
  const int h = blockIdx.x, b = blockIdx.y, slot = step.slot(b), len = step.len(b, a.S);
  if (slot < 0 || len <= 0) return;
  __shared__ float wf[4], wm[4];
  const size_t row = (size_t)b * a.H + h;
  u += row * a.P;
  r += row * a.P;
  m += row * (a.P + 1);
  if (PER) per = PER;
  const float bi = ld(bias + h), bf = ld(bias + a.H + h);
  const float m0 = step.first(b) ? state_m[(size_t)slot * a.H + h] : 0.f;
  const int t0 = threadIdx.x * per, t1 = min(t0 + per, a.P), lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  constexpr int NR = PER ? PER : 1;
  float i_of[NR], f_of[NR];
  auto gates = [&](int t, float zi, float zf, float& li, float& lf) {
    li = t < len ? log_input(zi, bi, a.cap) : -INFINITY;
    lf = t < len ? log_forget(zf, bf, a.cap) : 0.f;
  };
  auto inputs = [&](int t) { return proj + ((size_t)b * a.S + min(t, len - 1)) * a.N + h; };
  if (PER) {
#pragma unroll
    for (int k = 0; k < NR; ++k) {
      i_of[k] = ld(inputs(t0 + k) + a.i_at);
      f_of[k] = ld(inputs(t0 + k) + a.f_at);
    }
#pragma unroll
    for (int k = 0; k < NR; ++k) gates(t0 + k, i_of[k], f_of[k], i_of[k], f_of[k]);
  } else {
    for (int t = t0; t < t1; ++t) gates(t, ld(inputs(t) + a.i_at), ld(inputs(t) + a.f_at), r[t], u[t]);
  }
  // f(token, log input gate, log forget gate) for the thread's tokens
  auto walk = [&](auto f) {
    if (PER) {
#pragma unroll
      for (int k = 0; k < NR; ++k)
        if (t0 + k < t1) f(t0 + k, i_of[k], f_of[k]);
    } else
      for (int t = t0; t < t1; ++t) f(t, r[t], u[t]);
  };
  float F = 0.f, sf = 0.f, sm = -INFINITY;  // summed log forget gates, of the last chunk and in all; maximum
  walk([&](int t, float li, float lf) {
    if (t % C == 0) F = 0.f;
    F += lf;
    sf += lf;
    sm = fmaxf(sm + lf, li);
  });
  // summed forget gates of the chunk before this thread (threads of a chunk are neighbours)
  const int group = per >= C ? 1 : C / per;
  float before = F;
  for (int d = 1; d < group; d <<= 1) {
    const float o = __shfl_up(before, d);
    if ((lane & (group - 1)) >= d) before += o;
  }
  before = __shfl_up(before, 1);
  if ((lane & (group - 1)) == 0) before = 0.f;
  // maxima: (F, M) of a range followed by (F', M') is (F + F', max(M + F', M'))
  for (int d = 1; d < 64; d <<= 1) {
    const float of = __shfl_up(sf, d), om = __shfl_up(sm, d);
    if (lane >= d) { sm = fmaxf(om + sf, sm); sf += of; }
  }
  if (lane == 63) { wf[wave] = sf; wm[wave] = sm; }
  sf = __shfl_up(sf, 1);
  sm = __shfl_up(sm, 1);
  if (lane == 0) { sf = 0.f; sm = -INFINITY; }
  __syncthreads();
  float now = m0;
  for (int w = 0; w < wave; ++w) now = fmaxf(now + wf[w], wm[w]);
  now = fmaxf(now + sf, sm);
  if (threadIdx.x == 0) m[0] = m0;
  F = before;
  walk([&](int t, float li, float lf) {
    if (t % C == 0) F = 0.f;
    F += lf;
    now = fmaxf(now + lf, li);
    m[t + 1] = now;
    u[t] = F - now;
    r[t] = li - F;
    if (t == a.P - 1) state_m[(size_t)slot * a.H + h] = now;
  });
}

// operand of a product whose k runs over tiles of 16: a lane holds 4 of each
// tile at quad * 4, as it does of accumulators, so that these are operands too
template <typename T> DEVINL typename Frag<T>::V ld_tiles(const T* p);
template <> DEVINL bf16x8 ld_tiles<bf16_t>(const bf16_t* p) {
  union { bf16x8 v; ushort4_t h[2]; } f;
  f.h[0] = *(const ushort4_t*)p;
  f.h[1] = *(const ushort4_t*)(p + 16);
  return f.v;
}
template <> DEVINL floatx4 ld_tiles<float>(const float* p) { return *(const floatx4*)p; }

// fp32 numbers of one k step as operands: bf16 in two parts, fp32 as it is
template <typename T> struct Parts;
template <> struct Parts<bf16_t> {
  bf16x8 hi, lo;
  DEVINL void set(const floatx4* v) {
#pragma unroll
    for (int i = 0; i < 8; i += 2) {  // the upper halves as they are, and what they leave
      const unsigned x = __float_as_uint(v[i >> 2][i & 3]), y = __float_as_uint(v[i >> 2][(i & 3) + 1]);
      ((unsigned*)&hi)[i >> 1] = __builtin_amdgcn_perm(y, x, 0x07060302u);
      lo[i] = (__bf16)(__uint_as_float(x) - __uint_as_float(x & 0xffff0000u));
      lo[i + 1] = (__bf16)(__uint_as_float(y) - __uint_as_float(y & 0xffff0000u));
    }
  }
  static DEVINL floatx4 times(const Parts& x, const bf16x8& y, floatx4 c) { return mma(x.lo, y, mma(x.hi, y, c)); }
  static DEVINL floatx4 by(const bf16x8& y, const Parts& x, floatx4 c) { return mma(y, x.lo, mma(y, x.hi, c)); }
};
template <> struct Parts<float> {
  floatx4 x;
  DEVINL void set(const floatx4* v) { x = v[0]; }
  static DEVINL floatx4 times(const Parts& x, const floatx4& y, floatx4 c) { return mma(x.x, y, c); }
  static DEVINL floatx4 by(const floatx4& y, const Parts& x, floatx4 c) { return mma(y, x.x, c); }
};
DEVINL void to_floats(const bf16x8& f, floatx4* o) {
#pragma unroll
  for (int i = 0; i < 8; ++i) o[i >> 2][i & 3] = (float)f[i];
}
DEVINL void to_floats(const floatx4& f, floatx4* o) { o[0] = f; }

// WHOLE walks a row from its state to its end. Where rows are few and long, they
// are cut into segments: STATES walks each from zero and keeps its last state and
// decay, segment_kernel makes the state every segment starts from, OUTPUTS walks
// again from there.
enum Pass { WHOLE, STATES, OUTPUTS };

constexpr int ET = 2;  // tiles of 16 value channels that a wave owns

template <typename T, int DT> struct MemShape {
  static constexpr int DP = DT * 16;
  static constexpr int NP = 4;  // parts of the sum of keys, each of a share of the tokens
  static constexpr int PAD = sizeof(T) == 2 ? 8 : 4, QS = DP + PAD, CS = C + PAD;  // padded LDS rows
  static size_t lds(int waves, bool outputs) {
    size_t n = (size_t)(DP + waves * 32) * CS * sizeof(T) + (NP * DP + 4 * C) * sizeof(float);
    if (outputs) n += 2 * C * QS * sizeof(T) + (waves * 64 / C + waves + 1) * C * sizeof(float);
    return n;
  }
};

// four channels of four tokens, and the same by channel
template <typename T> struct Block4;
template <> struct Block4<bf16_t> {
  typedef ushort4_t Row;
  Row row[4];
  DEVINL void by_channel(Row* o) const {
    typedef __attribute__((ext_vector_type(2))) unsigned int uint2_t;
    uint2_t x[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) x[j] = __builtin_bit_cast(uint2_t, row[j]);
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const unsigned sel = i & 1 ? 0x07060302u : 0x05040100u;
      uint2_t v;
      v[0] = __builtin_amdgcn_perm(x[1][i >> 1], x[0][i >> 1], sel);
      v[1] = __builtin_amdgcn_perm(x[3][i >> 1], x[2][i >> 1], sel);
      o[i] = __builtin_bit_cast(Row, v);
    }
  }
};
template <> struct Block4<float> {
  typedef floatx4 Row;
  Row row[4];
  DEVINL void by_channel(Row* o) const {
#pragma unroll
    for (int i = 0; i < 4; ++i) o[i] = Row{row[0][i], row[1][i], row[2][i], row[3][i]};
  }
};

// One block per (segment, head, row), a wave per 32 value channels. A wave holds
// its channels of the state as accumulators, DT tiles of 16 key channels. VEC:
// addresses and widths allow loads and stores of four.
template <typename T, int DT, int PASS, bool VEC>
__global__ __launch_bounds__(512) void memory_kernel(
    const T* __restrict__ proj, const float* __restrict__ u, const float* __restrict__ r, const float* __restrict__ m,
    const T* __restrict__ norm, float* __restrict__ state, float* __restrict__ part, float* __restrict__ decay,
    T* __restrict__ out, MemArgs a, Step step) {
  typedef MemShape<T, DT> Sh;
  typedef typename Frag<T>::V V;
  typedef typename Block4<T>::Row Row;
  constexpr int DP = Sh::DP, QS = Sh::QS, CS = Sh::CS, KT = Frag<T>::K / 16;  // tiles of a k step
  constexpr int TT = C / 16, TG = C / 4;
  extern __shared__ __attribute__((aligned(16))) char mem[];
  const int TH = blockDim.x, waves = TH >> 6, EP = waves * 32, parts = TH / C;
  T* sKT = (T*)mem;             // [DP][CS] keys by channel
  T* sVT = sKT + DP * CS;       // [EP][CS] values by channel
  float* sn = (float*)(sVT + EP * CS);  // [NP][DP] the sum of keys
  float *su = sn + Sh::NP * DP, *sr = su + C, *sw = sr + C, *sa = sw + C;
  T* sQ = (T*)(sa + C);         // [C][QS]
  T* sK = sQ + C * QS;          // [C][QS]
  float* sdot = (float*)(sK + C * QS);  // [parts][C] queries with the sum of keys
  float* ssq = sdot + parts * C;        // [waves][C] squares of outputs
  float* srow = ssq + waves * C;        // [C] summed scores
  const int seg = blockIdx.x, h = blockIdx.y, b = blockIdx.z, tid = threadIdx.x;
  const int wave = tid >> 6, lane = tid & 63, col = lane & 15, quad = lane >> 4;
  const int slot = step.slot(b), len = slot < 0 ? 0 : step.len(b, a.S);
  const int c_lo = seg * a.seg, c_hi = min(c_lo + a.seg, a.P / C), c_end = min(c_hi, (len + C - 1) / C);
  const size_t head = (size_t)b * a.H + h;
  const float *ur = u + head * a.P, *rr = r + head * a.P, *mr = m + head * (a.P + 1);
  const T* rows = proj + (size_t)b * a.S * a.N;
  const int e0 = wave * 32;  // first value channel of this wave
  const size_t plane = (size_t)(a.vdim + 1) * a.dp;
  float* own = slot < 0 ? nullptr : state + ((size_t)slot * a.H + h) * plane;
  float* mine = PASS == WHOLE ? own : part + (((size_t)b * a.nseg + seg) * a.H + h) * plane;
  floatx4 S[DT][ET];
  const bool from_zero = PASS == STATES || (PASS == WHOLE && (slot < 0 || step.first(b) == 0)) || c_lo >= c_end;
#pragma unroll
  for (int i = 0; i < DT; ++i)
#pragma unroll
    for (int e = 0; e < ET; ++e) {
      const int c = e0 + e * 16 + col;
      S[i][e] = from_zero || c >= a.vdim || i * 16 >= a.dp ? (floatx4)(0.f)
                                                           : *(const floatx4*)(mine + (size_t)c * a.dp + i * 16 + quad * 4);
    }
  int np = 1;
  while (np < Sh::NP && np * 2 * DP <= TH) np *= 2;
  for (int d = tid; d < np * DP; d += TH) sn[d] = from_zero || d >= a.dp ? 0.f : mine[(size_t)a.vdim * a.dp + d];
  // the state is 2^held times the accumulators (and `sn`): while that does not get
  // too small, a chunk's decay goes there alone
  float log_decay = 0.f, held = 0.f;
  const float per_channel = 1.f / (float)a.vdim;
  float nw[ET][4];  // the norm's weights of this lane's outputs
#pragma unroll
  for (int e = 0; e < ET; ++e)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int c = e0 + e * 16 + quad * 4 + i;
      nw[e][i] = PASS != STATES && c < a.vdim ? ld(norm + h * a.vdim + c) * a.out_scale : 0.f;
    }
  // Channels c.. of token t0 + t + j; those past n hold others' numbers until
  // `within` clears them, which waits for the load. Tokens past the row's end are
  // read as its last: their weights are zero. In whole chunks a thread's places are
  // the same every time, apart from what is uniform.
  typedef __attribute__((ext_vector_type(sizeof(Row) / 4))) unsigned Bits;
  auto within = [](Row x, int c, int n) {
    if (VEC) return __builtin_bit_cast(Row, __builtin_bit_cast(Bits, x) & (c < n ? ~0u : 0u));
#pragma unroll
    for (int i = 0; i < 4; ++i)
      if (c + i >= n) x[i] = (T)0;
    return x;
  };
  auto fetch = [&](int t0, bool tail, int at, int t, int j, int c, int n) {
    Row x;
    if (VEC) {
      if (!tail) x = *(const Row*)((rows + (size_t)(t0 + j) * a.N + at) + (unsigned)(t * a.N + min(c, n - 4)));
      else x = *(const Row*)(rows + (size_t)min(t0 + t + j, len - 1) * a.N + at + min(c, n - 4));
    } else {
      const T* src = rows + (size_t)min(t0 + t + j, len - 1) * a.N + at;
#pragma unroll
      for (int i = 0; i < 4; ++i) x[i] = src[min(c + i, n - 1)];
    }
    return x;
  };
  // a block of four channels by four tokens: neighbouring lanes take 16
  // channels, then 8 tokens' blocks, which spreads LDS writes over all banks
  auto put = [&](const Block4<T>& x, int c, int t, T* by_col, T* by_row) {
    Row col4[4];
    x.by_channel(col4);
#pragma unroll
    for (int i = 0; i < 4; ++i) *(Row*)(by_col + (c + i) * CS + t) = col4[i];
    if (by_row)
#pragma unroll
      for (int j = 0; j < 4; ++j) *(Row*)(by_row + (t + j) * QS + c) = x.row[j];
  };
  // keys: DT * C blocks; queries: twice as many halves of them; values: a wave's own
  auto key_at = [&](int idx, int& c, int& t) {
    c = (idx & 3) * 4 + idx / C * 16;
    t = (idx >> 2) % TG * 4;
  };
  auto fetch_key = [&](int t0, bool tail, int idx, Block4<T>& k) {
    int c, t;
    key_at(idx, c, t);
#pragma unroll
    for (int j = 0; j < 4; ++j) k.row[j] = fetch(t0, tail, a.k_at + h * a.dim, t, j, c, a.dim);
  };
  auto put_key = [&](int idx, const Block4<T>& k) {
    int c, t;
    key_at(idx, c, t);
    if (idx < DT * C) put(k, c, t, sKT, PASS != STATES ? sK : (T*)nullptr);
  };
  auto fetch_query = [&](int t0, bool tail, int idx, Row* q) {
    const int t = min(idx / (DP / 8), C - 1);
#pragma unroll
    for (int j = 0; j < 2; ++j) q[j] = fetch(t0, tail, a.q_at + h * a.dim, t, 0, idx % (DP / 8) * 8 + j * 4, a.dim);
  };
  auto put_query = [&](int idx, const Row* q) {
    const int c = idx % (DP / 8) * 8;
#pragma unroll
    for (int j = 0; j < 2; ++j)
      if (idx < 2 * DT * C) *(Row*)(sQ + idx / (DP / 8) * QS + c + j * 4) = within(q[j], c + j * 4, a.dim);
  };
  const int vc = e0 + ((lane & 3) + (lane >> 5) * 4) * 4, vt = ((lane >> 2) & 7) * 4;
  // what a thread's first blocks of the next chunk hold, on its way while this one is computed
  constexpr int R = C / 32;
  Block4<T> k0[R], v0[R];
  Row q0[2 * R][2];
  float ut, rt, m_prev, u_last;
  auto ahead_of = [&](int t0, bool tail) {
#pragma unroll
    for (int i = 0; i < R; ++i) fetch_key(t0, tail, tid + i * TH, k0[i]);
#pragma unroll
    for (int i = 0; i < R; ++i)
#pragma unroll
      for (int j = 0; j < 4; ++j) v0[i].row[j] = fetch(t0, tail, a.v_at + h * a.vdim, i * 32 + vt, j, vc, a.vdim);
    if (PASS != STATES)
#pragma unroll
      for (int i = 0; i < 2 * R; ++i) fetch_query(t0, tail, tid + i * TH, q0[i]);
  };
  auto ahead = [&](int t0) {
    if (t0 + C > len) ahead_of(t0, true);
    else ahead_of(t0, false);
    ut = ur[t0 + tid % C];
    rt = rr[t0 + tid % C];
    m_prev = mr[t0];
    u_last = ur[t0 + C - 1];
  };
  if (c_lo < c_end) ahead(c_lo * C);
  for (int ch = c_lo; ch < c_end; ++ch) {
    const int t0 = ch * C;
    const bool tail = t0 + C > len;
    __syncthreads();  // everyone is done with the previous chunk
#pragma unroll
    for (int i = 0; i < R; ++i) {
      put_key(tid + i * TH, k0[i]);
#pragma unroll
      for (int j = 0; j < 4; ++j) v0[i].row[j] = within(v0[i].row[j], vc, a.vdim);
      put(v0[i], vc, i * 32 + vt, sVT, (T*)nullptr);
    }
    for (int idx = tid + R * TH; idx < DT * C; idx += TH) {
      Block4<T> k;
      fetch_key(t0, tail, idx, k);
      put_key(idx, k);
    }
    if (PASS != STATES) {
#pragma unroll
      for (int i = 0; i < 2 * R; ++i) put_query(tid + i * TH, q0[i]);
      for (int idx = tid + 2 * R * TH; idx < 2 * DT * C; idx += TH) {
        Row q[2];
        fetch_query(t0, tail, idx, q);
        put_query(idx, q);
      }
    }
    const float before = held;
    held += u_last + m_prev;
    log_decay += u_last + m_prev;
    const bool rescale = held < -20.f;
    const float whole = rescale ? pow2(held) : 1.f;
    if (rescale) held = 0.f;
    if (tid < C) {
      su[tid] = ut;
      sr[tid] = rt;
      sw[tid] = pow2(u_last + rt - held);
      sa[tid] = pow2(ut + m_prev + before) * a.scale;
    }
    __syncthreads();
    if (ch + 1 < c_end) ahead(t0 + C);
    if (PASS != STATES) {
      Row gate[TT][ET];
#pragma unroll
      for (int tt = 0; tt < TT; ++tt)
#pragma unroll
        for (int e = 0; e < ET; ++e) {
          gate[tt][e] = fetch(t0, tail, a.g_at + h * a.vdim, tt * 16 + col, 0, e0 + e * 16 + quad * 4, a.vdim);
        }
      {
        const int t = tid % C;
        float dot = 0.f;
        for (int d = tid / C * 4; d < DP; d += parts * 4) {
          floatx4 n = *(const floatx4*)(sn + d);
          for (int p = 1; p < np; ++p) n += *(const floatx4*)(sn + p * DP + d);
          float q[4];
          ld4(sQ + t * QS + d, q);
#pragma unroll
          for (int i = 0; i < 4; ++i) dot += n[i] * q[i];
        }
        sdot[tid] = dot;
      }
      constexpr bool HOLD = DT <= 8;  // queries' operands stay in registers
      V qf[HOLD ? TT : 1][HOLD ? DT / KT : 1];
      auto load_q = [&](int tt, int c) { return ld_tiles<T>(sQ + (tt * 16 + col) * QS + c * KT * 16 + quad * 4); };
      auto q_of = [&](int tt, int c) { return HOLD ? qf[HOLD ? tt : 0][HOLD ? c : 0] : load_q(tt, c); };
      if (HOLD)
#pragma unroll
        for (int tt = 0; tt < TT; ++tt)
#pragma unroll
          for (int c = 0; c < DT / KT; ++c) qf[HOLD ? tt : 0][HOLD ? c : 0] = load_q(tt, c);
      // what earlier chunks left
      floatx4 O[TT][ET];
#pragma unroll
      for (int tt = 0; tt < TT; ++tt)
#pragma unroll
        for (int e = 0; e < ET; ++e) O[tt][e] = (floatx4)(0.f);
#pragma unroll
      for (int c = 0; c < DT / KT; ++c)
#pragma unroll
        for (int e = 0; e < ET; ++e) {
          floatx4 s[KT];
#pragma unroll
          for (int k = 0; k < KT; ++k) s[k] = S[c * KT + k][e];
          Parts<T> p;
          p.set(s);
#pragma unroll
          for (int tt = 0; tt < TT; ++tt) O[tt][e] = Parts<T>::times(p, q_of(tt, c), O[tt][e]);
        }
      // scores of this chunk's tokens, keys by queries
      floatx4 w[TT][TT];
#pragma unroll
      for (int st = 0; st < TT; ++st)
#pragma unroll
        for (int tt = 0; tt < TT; ++tt) w[tt][st] = (floatx4)(0.f);
#pragma unroll
      for (int st = 0; st < TT; ++st)
#pragma unroll
        for (int c = 0; c < DT / KT; ++c) {
          const V kf = ld_tiles<T>(sK + (st * 16 + col) * QS + c * KT * 16 + quad * 4);
#pragma unroll
          for (int tt = st; tt < TT; ++tt) w[tt][st] = mma(kf, q_of(tt, c), w[tt][st]);
        }
      Parts<T> p[TT][TT / KT];
      float sum[TT];
#pragma unroll
      for (int tt = 0; tt < TT; ++tt) {
        const int t = tt * 16 + col;
        const float at = sa[t], here = su[t];
        sum[tt] = 0.f;
#pragma unroll
        for (int e = 0; e < ET; ++e) O[tt][e] *= at;
#pragma unroll
        for (int st = 0; st <= tt; ++st) {
          const floatx4 r4 = *(const floatx4*)(sr + st * 16 + quad * 4);
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            const float x = w[tt][st][i] * (a.scale * pow2(here + r4[i]));
            w[tt][st][i] = st < tt || quad * 4 + i <= col ? x : 0.f;
            sum[tt] += w[tt][st][i];
          }
        }
#pragma unroll
        for (int j = 0; j * KT <= tt; ++j) p[tt][j].set(&w[tt][j * KT]);
      }
#pragma unroll
      for (int j = 0; j < TT / KT; ++j)
#pragma unroll
        for (int e = 0; e < ET; ++e) {
          const V vf = ld_tiles<T>(sVT + (e0 + e * 16 + col) * CS + j * KT * 16 + quad * 4);
#pragma unroll
          for (int tt = j * KT; tt < TT; ++tt) O[tt][e] = Parts<T>::by(vf, p[tt][j], O[tt][e]);
        }
#pragma unroll
      for (int tt = 0; tt < TT; ++tt) {
        const int t = tt * 16 + col;
        float sq = 0.f;
#pragma unroll
        for (int e = 0; e < ET; ++e)
#pragma unroll
          for (int i = 0; i < 4; ++i) sq += O[tt][e][i] * O[tt][e][i];
        sq += __shfl_xor(sq, 16);
        sq += __shfl_xor(sq, 32);
        sum[tt] += __shfl_xor(sum[tt], 16);
        sum[tt] += __shfl_xor(sum[tt], 32);
        if (quad == 0) ssq[wave * C + t] = sq;
        if (quad == 0 && wave == 0) srow[t] = sum[tt];
      }
      __syncthreads();
#pragma unroll
      for (int tt = 0; tt < TT; ++tt) {
        const int t = tt * 16 + col;
        if (t0 + t >= a.S) continue;
        float dot = 0.f, sq = 0.f;
        for (int p = 0; p < parts; ++p) dot += sdot[p * C + t];
        for (int w = 0; w < waves; ++w) sq += ssq[w * C + t];
        const bool live = t0 + t < len;
        const float found = fabsf(srow[t] + sa[t] * dot);
        const float inv = __builtin_amdgcn_rcpf(fmaxf(found, pow2(live ? -mr[t0 + t + 1] : 0.f)) + 1e-6f);
        const float f = live ? inv * __builtin_amdgcn_rsqf(sq * inv * inv * per_channel + a.eps) : 0.f;
        T* dst = out + ((size_t)b * a.S + t0 + t) * a.K + a.out_at + h * a.vdim;
#pragma unroll
        for (int e = 0; e < ET; ++e) {
          const int c = e0 + e * 16 + quad * 4;
          if (c >= a.vdim) continue;
          float o[4];
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            T g = gate[tt][e][i];
            o[i] = O[tt][e][i] * f * nw[e][i] * sigmoidf(ld(&g));
          }
          if (VEC) st4(dst + c, o);
          else
#pragma unroll
            for (int i = 0; i < 4; ++i)
              if (c + i < a.vdim) st(dst + c + i, o[i]);
        }
      }
    }
    // the state after this chunk
    if (rescale)
#pragma unroll
      for (int i = 0; i < DT; ++i)
#pragma unroll
        for (int e = 0; e < ET; ++e) S[i][e] *= whole;
#pragma unroll
    for (int j = 0; j < TT / KT; ++j) {
      Parts<T> p[ET];
#pragma unroll
      for (int e = 0; e < ET; ++e) {
        floatx4 w[KT];
        to_floats(ld_tiles<T>(sVT + (e0 + e * 16 + col) * CS + j * KT * 16 + quad * 4), w);
#pragma unroll
        for (int k = 0; k < KT; ++k) w[k] *= *(const floatx4*)(sw + (j * KT + k) * 16 + quad * 4);
        p[e].set(w);
      }
#pragma unroll
      for (int i = 0; i < DT; ++i) {
        const V kf = ld_tiles<T>(sKT + (i * 16 + col) * CS + j * KT * 16 + quad * 4);
#pragma unroll
        for (int e = 0; e < ET; ++e) S[i][e] = Parts<T>::by(kf, p[e], S[i][e]);
      }
    }
    for (int i = tid; i < np * DP; i += TH) {
      const int d = i % DP, share = C / np, s0 = i / DP * share;
      float n = sn[i] * whole;
      for (int s = s0; s < s0 + share; s += 4) {
        float k[4], w[4];
        ld4(sKT + d * CS + s, k);
        ld4(sw + s, w);
#pragma unroll
        for (int i = 0; i < 4; ++i) n += k[i] * w[i];
      }
      sn[i] = n;
    }
  }
  // tokens past a row's end, and parked rows
  if (PASS != STATES)
    for (int t = max(c_lo, c_end) * C + wave; t < min(c_hi * C, a.S); t += waves)
      for (int c = lane; c < a.vdim; c += 64) st(out + ((size_t)b * a.S + t) * a.K + a.out_at + h * a.vdim + c, 0.f);
  if (PASS == OUTPUTS || len <= 0) return;
  const float scale = pow2(held);
  if (PASS == STATES && tid == 0) decay[((size_t)b * a.nseg + seg) * a.H + h] = pow2(log_decay);
#pragma unroll
  for (int i = 0; i < DT; ++i)
#pragma unroll
    for (int e = 0; e < ET; ++e) {
      const int c = e0 + e * 16 + col;
      if (c < a.vdim && i * 16 < a.dp) *(floatx4*)(mine + (size_t)c * a.dp + i * 16 + quad * 4) = S[i][e] * scale;
    }
  __syncthreads();
  for (int d = tid; d < a.dp; d += TH) {
    float n = sn[d];
    for (int p = 1; p < np; ++p) n += sn[p * DP + d];
    mine[(size_t)a.vdim * a.dp + d] = n * scale;
  }
}

// part [B][nseg][H][..]: every segment's own last state -> the state it starts
// from; state: that after the row
__global__ __launch_bounds__(256) void segment_kernel(float* __restrict__ part, const float* __restrict__ decay,
                                                      float* __restrict__ state, int plane, MemArgs a, Step step) {
  const int i = (blockIdx.x * 256 + threadIdx.x) * 4, h = blockIdx.y, b = blockIdx.z, slot = step.slot(b);
  if (i >= plane || slot < 0 || step.len(b, a.S) <= 0) return;
  floatx4* own = (floatx4*)(state + ((size_t)slot * a.H + h) * plane + i);
  floatx4 now = step.first(b) ? *own : (floatx4)(0.f);
  const size_t stride = (size_t)a.H * plane;
  float* p = part + ((size_t)b * a.nseg * a.H + h) * plane + i;
  constexpr int AHEAD = 8;
  for (int s0 = 0; s0 < a.nseg; s0 += AHEAD) {
    floatx4 x[AHEAD];
    float d[AHEAD];
#pragma unroll
    for (int j = 0; j < AHEAD; ++j)
      if (s0 + j < a.nseg) {
        x[j] = *(const floatx4*)(p + (s0 + j) * stride);
        d[j] = decay[((size_t)b * a.nseg + s0 + j) * a.H + h];
      }
#pragma unroll
    for (int j = 0; j < AHEAD; ++j)
      if (s0 + j < a.nseg) {
        *(floatx4*)(p + (s0 + j) * stride) = now;
        now = now * d[j] + x[j];
      }
  }
  *own = now;
}

// Decode: one block per (head, row); 16 lanes share a column of the state, RPL
// key channels each.
template <int RPL> struct Rows {
  static constexpr int V = RPL % 4 == 0 ? 4 : RPL % 2 == 0 ? 2 : 1;
  static DEVINL int at(int j, int r) { return j * 16 * V + V * r; }
};
template <int V>
DEVINL void ld_any(const float* p, float* o) {
  if (V == 4) ld4(p, o);
  else if (V == 2) ld2(p, o);
  else o[0] = *p;
}
template <int V>
DEVINL void st_any(float* p, const float* o) {
  if (V == 4) st4(p, o);
  else if (V == 2) st2(p, o);
  else *p = o[0];
}

template <typename T, int RPL>
__global__ __launch_bounds__(256) void memory_step_kernel(const T* __restrict__ proj, const T* __restrict__ bias,
                                                          const T* __restrict__ norm, float* __restrict__ state,
                                                          float* __restrict__ state_m, T* __restrict__ out, MemArgs a,
                                                          Step step) {
  constexpr int DP = 16 * RPL, NB = RPL <= 8 ? 8 : 4, VW = Rows<RPL>::V;  // NB: columns in flight per 16 lanes
  __shared__ __attribute__((aligned(16))) float sq[DP], sk[DP];
  __shared__ float so[256], red[4], sfound;
  const int h = blockIdx.x, b = blockIdx.y, tid = threadIdx.x, slot = step.slot(b);
  T* dst = out + (size_t)b * a.K + a.out_at + h * a.vdim;
  if (slot < 0) {
    if (tid < a.vdim) st(dst + tid, 0.f);
    return;
  }
  const int pos = step.first(b), r = tid & 15, cl = tid >> 4;
  const T* row = proj + (size_t)b * a.N;
  float* base = state + ((size_t)slot * a.H + h) * (size_t)(a.vdim + 1) * DP;
  float s[NB][RPL], v[NB], n[RPL];
  auto load = [&](int c0) {
#pragma unroll
    for (int i = 0; i < NB; ++i) {
      const int c = min(c0 + i * 16 + cl, a.vdim - 1);
      v[i] = ld(row + a.v_at + h * a.vdim + c);
#pragma unroll
      for (int j = 0; j < RPL / VW; ++j) ld_any<VW>(base + (size_t)c * DP + Rows<RPL>::at(j, r), s[i] + j * VW);
    }
  };
  load(0);  // in flight while the gates are made
#pragma unroll
  for (int j = 0; j < RPL / VW; ++j) ld_any<VW>(base + (size_t)a.vdim * DP + Rows<RPL>::at(j, r), n + j * VW);
  if (tid < DP) {
    sq[tid] = tid < a.dim ? ld(row + a.q_at + h * a.dim + tid) * a.scale : 0.f;
    sk[tid] = tid < a.dim ? ld(row + a.k_at + h * a.dim + tid) : 0.f;
  }
  float* mp = state_m + (size_t)slot * a.H + h;
  const float li = log_input(ld(row + a.i_at + h), ld(bias + h), a.cap);
  const float lf = log_forget(ld(row + a.f_at + h), ld(bias + a.H + h), a.cap);
  const float m0 = pos > 0 ? *mp : 0.f, top = fmaxf(lf + m0, li);
  const float keep = pow2(lf + m0 - top), take = pow2(li - top);
  float gate = 0.f, weight = 0.f;
  if (tid < a.vdim) {
    gate = ld(row + a.g_at + h * a.vdim + tid);
    weight = ld(norm + h * a.vdim + tid);
  }
  __syncthreads();
  if (tid == 0) *mp = top;  // everyone has read it
  float q[RPL], k[RPL];
#pragma unroll
  for (int j = 0; j < RPL / VW; ++j) {
    ld_any<VW>(sq + Rows<RPL>::at(j, r), q + j * VW);
    ld_any<VW>(sk + Rows<RPL>::at(j, r), k + j * VW);
  }
#pragma unroll
  for (int i = 0; i < RPL; ++i) k[i] *= take;
  // a row of 16 channels of one column; what a new sequence's slot held does not count
  auto advance = [&](float* x, float value, float* to) {
    float o = 0.f;
#pragma unroll
    for (int j = 0; j < RPL; ++j) {
      x[j] = (pos > 0 ? keep * x[j] : 0.f) + k[j] * value;
      o += x[j] * q[j];
    }
    if (to)
#pragma unroll
      for (int j = 0; j < RPL / VW; ++j) st_any<VW>(to + Rows<RPL>::at(j, r), x + j * VW);
    return row_sum(o);
  };
  for (int c0 = 0; c0 < a.vdim; c0 += 16 * NB) {
    if (c0) load(c0);
#pragma unroll
    for (int i = 0; i < NB; ++i) {
      const int c = c0 + i * 16 + cl;
      const float o = advance(s[i], v[i], c < a.vdim ? base + (size_t)c * DP : nullptr);
      if (r == 0 && c < a.vdim) so[c] = o;
    }
  }
  __syncthreads();  // every wave has read the sum of keys
  const float found = advance(n, 1.f, cl == 0 ? base + (size_t)a.vdim * DP : nullptr);
  if (tid == 0) sfound = fabsf(found);
  __syncthreads();
  const float inv = 1.f / (fmaxf(sfound, pow2(-top)) + 1e-6f);
  const float y = tid < a.vdim ? so[tid] * inv : 0.f;
  const float f = 1.f / sqrtf(block_sum(y * y, red) / (float)a.vdim + a.eps) * a.out_scale;
  if (tid < a.vdim) st(dst + tid, y * f * weight * sigmoidf(gate));
}

// ===========================================================================
// host side
// ===========================================================================

static int row_pad(int dim) {
  for (int p : {1, 2, 3, 4, 6, 8, 12, 16})
    if (dim <= 16 * p) return 16 * p;
  TORCH_CHECK(false, "a memory of ", dim, " key channels (at most 256)");
}

template <typename T, int DT>
static void prompt(const Tensor& proj, const Tensor& u, const Tensor& r, const Tensor& m, const Tensor& norm,
                   Tensor& state, Tensor& out, int B, MemArgs a, const Step& step) {
  typedef MemShape<T, DT> Sh;
  const int waves = (a.vdim + 31) / 32, chunks = a.P / C, plane = (a.vdim + 1) * a.dp;
  // rows are cut while the chip's 256 units do not have two blocks each; a
  // segment is worth its second walk from eight chunks on
  const int want = (512 + B * a.H - 1) / (B * a.H), most = std::max(1, chunks / 8);
  a.seg = (chunks + std::min(want, most) - 1) / std::min(want, most);
  a.nseg = (chunks + a.seg - 1) / a.seg;
  TORCH_CHECK(B <= 65535 && a.H <= 65535, "a prefill step of ", B, " rows and ", a.H, " heads is too large");
  const hipStream_t stream = cur_stream();
  Tensor part, decay;
  if (a.nseg > 1) {
    part = f32(proj, {B, a.nseg, a.H, plane});
    decay = f32(proj, {B, a.nseg, a.H});
  }
  float *pp = a.nseg > 1 ? M<float>(part) : nullptr, *dp = a.nseg > 1 ? M<float>(decay) : nullptr;
  const bool vec = ((a.dim | a.vdim | a.N | a.q_at | a.k_at | a.v_at | a.g_at | a.K | a.out_at) & 3) == 0;
  if (!vec) { a.seg = chunks; a.nseg = 1; }
  auto run = [&](auto kernel, bool outputs) {
    static const hipError_t err = hipFuncSetAttribute((const void*)kernel, hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
    TORCH_CHECK(err == hipSuccess, "no LDS for the memory's chunks");
    const size_t lds = Sh::lds(waves, outputs);
    TORCH_CHECK(lds <= 160 * 1024, "a memory of ", a.dim, " by ", a.vdim, " channels does not fit LDS");
    hipLaunchKernelGGL(kernel, dim3(a.nseg, a.H, B), dim3(64 * waves), lds, stream, P<T>(proj), P<float>(u), P<float>(r),
                       P<float>(m), P<T>(norm), M<float>(state), pp, dp, M<T>(out), a, step);
  };
  if (!vec) { run(memory_kernel<T, DT, WHOLE, false>, true); return; }
  if (a.nseg == 1) { run(memory_kernel<T, DT, WHOLE, true>, true); return; }
  run(memory_kernel<T, DT, STATES, true>, false);
  hipLaunchKernelGGL(segment_kernel, dim3((plane / 4 + 255) / 256, a.H, B), dim3(256), 0, stream, pp, dp, M<float>(state),
                     plane, a, step);
  run(memory_kernel<T, DT, OUTPUTS, true>, true);
}

// proj [B,S,N]; bias [2,H] of input and forget gate; state [slots,H,vdim+1,dp]
// (the last row sums the keys), state_m [slots,H]
void matrix_memory(Tensor proj, int64_t q_at, int64_t k_at, int64_t v_at, int64_t g_at, int64_t i_at, int64_t f_at,
                   int64_t H, int64_t dim, int64_t vdim, Tensor bias, double cap, Tensor norm, double eps, Tensor state,
                   Tensor state_m, OptT slots, OptT positions, OptT lens, int64_t start, bool decode, Tensor out,
                   int64_t out_at, double out_scale) {
  const auto dt = io_type(proj);
  for (const Tensor& t : {bias, norm, out}) check_io(t, dt);
  check_io(state, torch::kFloat32);
  check_io(state_m, torch::kFloat32);
  CHK(proj.dim() == 3 && out.dim() == 3 && out.size(0) == proj.size(0) && out.size(1) == proj.size(1));
  const int B = proj.size(0), S = proj.size(1), N = proj.size(2), dp = row_pad(dim);
  CHK(H > 0 && dim > 0 && vdim > 0 && cap > 0);
  TORCH_CHECK(vdim <= 256, "a memory of ", vdim, " value channels (at most 256)");
  for (int64_t at : {q_at, k_at}) CHK(at >= 0 && at + H * dim <= N);
  for (int64_t at : {v_at, g_at}) CHK(at >= 0 && at + H * vdim <= N);
  CHK(i_at >= 0 && i_at + H <= N && f_at >= 0 && f_at + H <= N && out_at >= 0 && out_at + H * vdim <= out.size(2));
  CHK(bias.numel() == 2 * H && norm.numel() == H * vdim && (!decode || S == 1));
  CHK(state.dim() == 4 && state.size(1) == H && state.size(2) == vdim + 1 && state.size(3) == dp);
  CHK(state_m.dim() == 2 && state_m.size(0) == state.size(0) && state_m.size(1) == H && (slots || B <= state.size(0)));
  if (B == 0 || S == 0) return;
  const Step step = make_step(slots, positions, lens, start, decode, B);
  MemArgs a{S, (int)H, N, (int)out.size(2), (int)q_at, (int)k_at, (int)v_at, (int)g_at, (int)i_at, (int)f_at, (int)out_at,
            (int)dim, (int)vdim, dp, 0, 0, 0, (float)cap, (float)eps, 1.f / sqrtf((float)dim), (float)out_scale};
  const hipStream_t stream = cur_stream();
  if (decode) {
#define STEP(R)                                                                                                    \
  case R: hipLaunchKernelGGL((memory_step_kernel<T, R>), dim3(H, B), dim3(256), 0, stream, P<T>(proj), P<T>(bias), \
                             P<T>(norm), M<float>(state), M<float>(state_m), M<T>(out), a, step);                  \
    break
    BY_TYPE(dt, {
      switch (dp / 16) { STEP(1); STEP(2); STEP(3); STEP(4); STEP(6); STEP(8); STEP(12); STEP(16); }
    });
#undef STEP
    return;
  }
  BY_TYPE(dt, {
    a.P = (S + C - 1) / C * C;
    auto u = f32(proj, {B, H, a.P}), r = f32(proj, {B, H, a.P}), m = f32(proj, {B, H, a.P + 1});
    int per = 1;
    while (per * 256 < a.P) per *= 2;
    auto gates = [&](auto kernel) {
      hipLaunchKernelGGL(kernel, dim3(H, B), dim3(256), 0, stream, P<T>(proj), P<T>(bias), M<float>(state_m), M<float>(u),
                         M<float>(r), M<float>(m), per, a, step);
    };
    if (per == 1) gates(gates_kernel<T, 1>);
    else if (per <= 4) { per = 4; gates(gates_kernel<T, 4>); }
    else if (per <= 16) { per = 16; gates(gates_kernel<T, 16>); }
    else gates(gates_kernel<T, 0>);
    if (dp <= 32) prompt<T, 2>(proj, u, r, m, norm, state, out, B, a, step);
    else if (dp <= 64) prompt<T, 4>(proj, u, r, m, norm, state, out, B, a, step);
    else if (dp <= 128) prompt<T, 8>(proj, u, r, m, norm, state, out, B, a, step);
    else prompt<T, 16>(proj, u, r, m, norm, state, out, B, a, step);
  });
}

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.def("matrix_memory", &matrix_memory, "matrix memory with exponential gates, per-head norm and output gate");
}
