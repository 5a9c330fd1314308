// CDNA4 (gfx950) kernels around an fp32 residual stream whose layers hand on
// averages over depth:
//   - embedding of tokens and of token pairs
//   - a layer's end in one pass: stream + its sublayers' outputs joins the
//     streams so far, their weighted sum is the new stream, which is RMS-normed
//     with one number per reader; in a decode step the first reader's causal
//     convolution too
//   - gelu_tanh(gate) * up on a packed projection; cap * tanh(x / cap)
//
// Two element types, bf16 and fp32; streams, norms and sums are fp32 in both.
// Rows of a step address state by slot (struct Step): slot -1 is a parked row,
// which reads and writes no state. A row at position 0 ignores what its slot
// holds.

#include "common.h"

// ---------------------------------------------------------------------------
// embedding
// ---------------------------------------------------------------------------

struct PairRule { long long buckets, mul_prev, mul_cur; };

// One block per token. last [slots]: the token before a row's step; the block of
// the first token reads it and leaves the row's last one.
template <typename T, int V>
__global__ __launch_bounds__(256) void embed_pairs_kernel(
    const long long* __restrict__ tokens, const T* __restrict__ table, const T* __restrict__ pairs,
    int* __restrict__ last, float* __restrict__ x, int S, int D, float scale, PairRule rule, Step step) {
  const int s = blockIdx.x, b = blockIdx.y, slot = step.slot(b), len = step.decode ? 1 : step.len(b, S);
  const long long* row = tokens + (size_t)b * S;
  const long long cur = row[s];
  long long prev = -1;
  if (s > 0) prev = row[s - 1];
  else if (slot >= 0 && len > 0) {
    if (last && step.first(b) > 0) prev = last[slot];
    __syncthreads();
    if (last && threadIdx.x == 0) last[slot] = (int)row[len - 1];
  }
  long long at = rule.buckets;
  if (prev >= 0) {
    at = (prev * rule.mul_prev + cur * rule.mul_cur) % rule.buckets;
    if (at < 0) at += rule.buckets;
  }
  const T *e = table + cur * D, *p = pairs + at * D;
  float* dst = x + ((size_t)b * S + s) * D;
  for (int i = threadIdx.x * V; i < D; i += 256 * V) {
    float a[V], c[V];
    ldv<V>(e + i, a);
    ldv<V>(p + i, c);
#pragma unroll
    for (int j = 0; j < V; ++j) a[j] = a[j] * scale + c[j];
    stv<V>(dst + i, a);
  }
}

// ---------------------------------------------------------------------------
// a layer's end
// ---------------------------------------------------------------------------

struct DepthArgs {
  int D, top, zs, done, taps;  // width; rows of z a token sums (0: its own), their stride; streams so far
  size_t plane;                // elements of one stream
  float eps;
};

template <typename T> DEVINL float rounded(float f) { return f; }
template <> DEVINL float rounded<bf16_t>(float f) { bf16_t u = f2b(f); return ld(&u); }

// One block per token; its row stays in registers (NC pieces of TB V). y null:
// x is read as it is; x null: it is the average with `before`. streams [done +
// 1][tokens][D]: the last one is written here. out null: nobody reads it. h1 = norm(x) g1, h2 = norm(x) g2, the first plus its convolution if
// there are taps. Loads that hang on nothing come first: one token's blocks are
// all that a decode step of few rows has.
template <typename T, int V, int NC, int TB>
__global__ __launch_bounds__(TB) void depth_norm_kernel(
    const T* __restrict__ y, const T* __restrict__ z, const int* __restrict__ rows, const float* __restrict__ weight,
    const float* __restrict__ x, float* __restrict__ streams, const T* __restrict__ before,
    const T* __restrict__ average, float* __restrict__ out, const T* __restrict__ g1, const T* __restrict__ g2,
    const T* __restrict__ taps, T* __restrict__ ring, T* __restrict__ h1, T* __restrict__ h2, DepthArgs a, Step step) {
  const size_t tok = blockIdx.x, off = tok * a.D;
  __shared__ float red[TB / 64];
  constexpr int BACK = NC <= 2 ? 3 : 0;  // inputs of the convolution in registers
  const int slot = taps ? step.slot((int)tok) : -1, pos = slot >= 0 ? step.first((int)tok) : 0;
  T* hist = ring + (size_t)max(slot, 0) * a.taps * a.D;
  float old[BACK + 1][NC * V];
#pragma unroll
  for (int k = 0; k < BACK; ++k)
#pragma unroll
    for (int c = 0; c < NC; ++c) {
      const int i = (c * TB + threadIdx.x) * V;
#pragma unroll
      for (int j = 0; j < V; ++j) old[k][c * V + j] = 0.f;
      if (slot >= 0 && k + 1 < a.taps && k + 1 <= pos && i < a.D)
        ldv<V>(hist + (size_t)((pos - 1 - k) % a.taps) * a.D + i, old[k] + c * V);
    }
  const float n1 = g1 ? ld(g1) : 0.f, n2 = g2 ? ld(g2) : 0.f;
  // a lane has the weights of one stream of 64
  const int lane = threadIdx.x & 63;
  auto lane_weight = [&](const T* w, int n0, int count) { return w && n0 + lane < count ? ld(w + n0 + lane) : 0.f; };
  auto of_lane = [](float w, int n) { return __uint_as_float(__builtin_amdgcn_readlane(__float_as_uint(w), n & 63)); };
  const float first_now = lane_weight(average, 0, a.done), first_before = lane_weight(before, 0, a.done);
  const float last = average ? ld(average + a.done) : 0.f;
  float xv[NC * V], ss = 0.f;
#pragma unroll
  for (int c = 0; c < NC; ++c) {
    const int at = (c * TB + threadIdx.x) * V, i = min(at, a.D - V);  // all lanes go along: weights are theirs
    float* v = xv + c * V;
#pragma unroll
    for (int j = 0; j < V; ++j) v[j] = 0.f;
    if (x) ldv<V>(x + off + i, v);
    if (y) {
      float sum[V], t[V];
#pragma unroll
      for (int j = 0; j < V; ++j) sum[j] = 0.f;
      const float* s = streams + off + i;
      float now = first_now, then = first_before;
      auto add = [&](int n, auto count) {  // `count` streams from n on, loads first
        constexpr int N = decltype(count)::value;
        float u[N][V];
#pragma unroll
        for (int k = 0; k < N; ++k) ldv<V>(s + (n + k) * a.plane, u[k]);
        if (n && (n & 63) == 0) {
          now = lane_weight(average, n, a.done);
          then = lane_weight(before, n, a.done);
        }
#pragma unroll
        for (int k = 0; k < N; ++k) {
          const float w = of_lane(now, n + k), p = of_lane(then, n + k);
#pragma unroll
          for (int j = 0; j < V; ++j) {
            sum[j] += w * u[k][j];
            v[j] += p * u[k][j];
          }
        }
      };
      ldv<V>(y + off + i, t);
#pragma unroll
      for (int j = 0; j < V; ++j) v[j] += t[j];
      if (z && !rows) {
        ldv<V>(z + tok * a.zs + i, t);
#pragma unroll
        for (int j = 0; j < V; ++j) v[j] += t[j];
      }
#pragma unroll 4
      for (int k = 0; k < a.top; ++k) {
        const float w = weight ? weight[tok * a.top + k] : 1.f;
        ldv<V>(z + (size_t)rows[tok * a.top + k] * a.zs + i, t);
#pragma unroll
        for (int j = 0; j < V; ++j) v[j] += w * t[j];
      }
      int n = 0;
      for (; n + 8 <= a.done; n += 8) add(n, std::integral_constant<int, 8>());
      if (n + 4 <= a.done) { add(n, std::integral_constant<int, 4>()); n += 4; }
      if (n + 2 <= a.done) { add(n, std::integral_constant<int, 2>()); n += 2; }
      if (n < a.done) add(n, std::integral_constant<int, 1>());
      if (at < a.D) stv<V>(streams + a.done * a.plane + off + i, v);
#pragma unroll
      for (int j = 0; j < V; ++j) v[j] = sum[j] + last * v[j];
      if (out && at < a.D) stv<V>(out + off + i, v);
    }
#pragma unroll
    for (int j = 0; j < V; ++j) ss += at < a.D ? v[j] * v[j] : 0.f;
  }
  if (!g1) return;
  ss = wave_sum(ss);
  if (lane == 0) red[threadIdx.x >> 6] = ss;
  __syncthreads();
  ss = 0.f;
#pragma unroll
  for (int w = 0; w < TB / 64; ++w) ss += red[w];
  const float inv = 1.f / sqrtf(ss / (float)a.D + a.eps);
  const float f1 = inv * n1, f2 = inv * n2;
#pragma unroll
  for (int c = 0; c < NC; ++c) {
    const int i = (c * TB + threadIdx.x) * V;
    if (i >= a.D) continue;
    float o[V];
#pragma unroll
    for (int j = 0; j < V; ++j) o[j] = rounded<T>(xv[c * V + j] * f1);
    if (slot >= 0) {
      stv<V>(hist + (size_t)(pos % a.taps) * a.D + i, o);  // the oldest input: no tap reaches it any more
      const T* w = taps + (size_t)i * a.taps + a.taps - 1;
      float sum[V];
#pragma unroll
      for (int j = 0; j < V; ++j) sum[j] = o[j] + o[j] * ld(w + j * a.taps);
#pragma unroll
      for (int k = 0; k < BACK; ++k)
        if (k + 1 < a.taps)
#pragma unroll
          for (int j = 0; j < V; ++j) sum[j] += old[k][c * V + j] * ld(w + j * a.taps - 1 - k);
      for (int back = min(a.taps - 1, pos); back > BACK; --back) {
        float t[V];
        ldv<V>(hist + (size_t)((pos - back) % a.taps) * a.D + i, t);
#pragma unroll
        for (int j = 0; j < V; ++j) sum[j] += t[j] * ld(w + j * a.taps - back);
      }
#pragma unroll
      for (int j = 0; j < V; ++j) o[j] = sum[j];
    }
    stv<V>(h1 + off + i, o);
    if (g2) {
#pragma unroll
      for (int j = 0; j < V; ++j) o[j] = xv[c * V + j] * f2;
      stv<V>(h2 + off + i, o);
    }
  }
}

// ---------------------------------------------------------------------------
// elementwise
// ---------------------------------------------------------------------------

template <typename T, int V>
__global__ __launch_bounds__(256) void geglu_kernel(const T* __restrict__ gu, T* __restrict__ out, long long n, int I) {
  const long long i = ((long long)blockIdx.x * 256 + threadIdx.x) * V;
  if (i >= n) return;
  const long long row = i / I;
  const int c = (int)(i - row * I);
  float g[V], u[V];
  ldv<V>(gu + row * 2 * I + c, g);
  ldv<V>(gu + row * 2 * I + I + c, u);
#pragma unroll
  for (int j = 0; j < V; ++j) u[j] *= gelu_tanh(g[j]);
  stv<V>(out + i, u);
}

template <typename T, int V>
__global__ __launch_bounds__(256) void soft_cap_kernel(const T* __restrict__ x, float* __restrict__ out, long long n,
                                                       float cap) {
  const long long i = ((long long)blockIdx.x * 256 + threadIdx.x) * V;
  if (i >= n) return;
  float v[V];
  ldv<V>(x + i, v);
#pragma unroll
  for (int j = 0; j < V; ++j) v[j] = cap * tanhf(v[j] / cap);
  stv<V>(out + i, v);
}

// ===========================================================================
// host side
// ===========================================================================

// tokens [B,S]; table [vocab,D]; pairs [buckets + 1,D]; last [slots,1] or none
void embed_pairs(Tensor tokens, Tensor table, double scale, Tensor pairs, int64_t buckets, int64_t mul_prev,
                 int64_t mul_cur, OptT last, OptT slots, OptT positions, OptT lens, int64_t start, bool decode, Tensor x) {
  const auto dt = io_type(table);
  check_io(pairs, dt);
  check_io(x, torch::kFloat32);
  tokens = tokens.to(torch::kInt64).contiguous();
  CHK(tokens.is_cuda() && tokens.dim() == 2 && table.dim() == 2 && pairs.dim() == 2);
  const int B = tokens.size(0), S = tokens.size(1), D = table.size(1);
  CHK(buckets > 0 && pairs.size(0) == buckets + 1 && pairs.size(1) == D && x.numel() == (int64_t)B * S * D);
  CHK((!decode || S == 1) && B <= 65535);
  if (last) { check_io(*last, torch::kInt32); CHK(last->dim() == 2 && last->size(1) == 1 && (slots || B <= last->size(0))); }
  if (B == 0 || S == 0) return;
  const Step step = make_step(slots, positions, lens, start, decode, B);
  const PairRule rule{buckets, mul_prev, mul_cur};
#define EMBED(V)                                                                                                      \
  hipLaunchKernelGGL((embed_pairs_kernel<T, V>), dim3(S, B), dim3(256), 0, cur_stream(),                              \
                     (const long long*)tokens.data_ptr<int64_t>(), P<T>(table), P<T>(pairs),                         \
                     last ? last->data_ptr<int>() : nullptr, M<float>(x), S, D, (float)scale, rule, step)
  BY_TYPE(dt, {
    if (D % 4 == 0) EMBED(4);
    else EMBED(1);
  });
#undef EMBED
}

// y [tokens,D] (none: x is read as it is), z the same, or with rows (and weight)
// [tokens,top] rows that a token sums; streams [n,..,D], of which `done` are
// filled; x [..,D], or before [done]: it is their average with these weights;
// average [done + 1]. -> (new stream if `keep`, h1, h2)
std::vector<OptT> depth_norm(OptT y, OptT z, OptT rows, OptT weight, OptT x, OptT before, OptT streams, int64_t done,
                             OptT average, bool keep, OptT g1, OptT g2, OptT taps, OptT ring, OptT slots, OptT positions,
                             double eps, bool bf16) {
  const auto dt = bf16 ? torch::kBFloat16 : torch::kFloat32;
  CHK(y ? (bool)streams : x && !z && !streams);
  if (x) check_io(*x, torch::kFloat32);
  if (streams) check_io(*streams, torch::kFloat32);
  const Tensor like = x ? *x : (*streams)[0];
  const int D = like.size(-1), n = like.numel() / D;
  DepthArgs a{D, 0, D, (int)done, 0, (size_t)like.numel(), (float)eps};
  if (y) {
    check_io(*y, dt);
    CHK(y->numel() == like.numel() && average && (bool)x != (bool)before);
    check_io(*average, dt);
    CHK(done >= 0 && streams->size(0) > done && streams->numel() == streams->size(0) * like.numel());
    CHK(average->numel() == done + 1);
  }
  if (before) { check_io(*before, dt); CHK(y && before->numel() == done); }
  if (z) {
    check_io(*z, dt);
    a.zs = z->size(-1);
    if (rows) {
      check_io(*rows, torch::kInt32);
      a.top = rows->size(-1);
      CHK(rows->numel() == (int64_t)n * a.top && z->numel() == rows->numel() * a.zs && a.zs >= D);
    } else CHK(z->numel() == like.numel() && a.zs == D);
  } else CHK(!rows && !weight);
  if (weight) { check_io(*weight, torch::kFloat32); CHK(rows && weight->numel() == rows->numel()); }
  CHK((g1 || !g2) && (g1 || !taps));
  if (g1) { check_io(*g1, dt); CHK(g1->numel() == 1); }
  if (g2) { check_io(*g2, dt); CHK(g2->numel() == 1); }
  Step step{};
  if (taps) {
    check_io(*taps, dt);
    CHK(ring && taps->dim() == 2 && taps->size(0) == D && taps->size(1) >= 1);
    check_io(*ring, dt);
    a.taps = taps->size(1);
    CHK(ring->dim() == 3 && ring->size(1) == a.taps && ring->size(2) == D && (slots || n <= ring->size(0)));
    step = make_step(slots, positions, c10::nullopt, 0, true, n);
  }
  const auto io = like.options().dtype(dt);
  OptT out, h1, h2;
  if (y && keep) out = torch::empty_like(like);
  if (g1) h1 = torch::empty(like.sizes(), io);
  if (g2) h2 = torch::empty(like.sizes(), io);
  if (n == 0) return {out, h1, h2};
#define AT(TYPE, t) (t ? (TYPE*)t->data_ptr() : nullptr)
#define NORM(V, NC, TB)                                                                                               \
  if (nc <= NC) {                                                                                                     \
    hipLaunchKernelGGL((depth_norm_kernel<T, V, NC, TB>), dim3(n), dim3(TB), 0, cur_stream(), AT(const T, y), AT(const T, z), \
                       AT(const int, rows), AT(const float, weight), AT(const float, x), AT(float, streams),          \
                       AT(const T, before), AT(const T, average), AT(float, out), AT(const T, g1), AT(const T, g2), AT(const T, taps),     \
                       AT(T, ring), AT(T, h1), AT(T, h2), a, step);                                                   \
    return {out, h1, h2};                                                                                             \
  }
  BY_TYPE(dt, {
    if (((D | a.zs) & 3) == 0) {
      if (n <= 256 && D > 1024) {  // few tokens: a row over more waves
        const int nc = (D + 4095) / 4096;
        if (D <= 2048) NORM(4, 1, 512)
        NORM(4, 1, 1024) NORM(4, 2, 1024) NORM(4, 4, 1024)
      }
      const int nc = (D + 1023) / 1024;
      NORM(4, 1, 256) NORM(4, 2, 256) NORM(4, 4, 256) NORM(4, 8, 256) NORM(4, 16, 256)
    } else {
      const int nc = (D + 255) / 256;
      NORM(1, 1, 256) NORM(1, 4, 256) NORM(1, 16, 256)
    }
  });
#undef NORM
#undef AT
  TORCH_CHECK(false, "row of ", D, " elements is too long");
}

Tensor geglu_packed(Tensor gu) {
  const auto dt = io_type(gu);
  const int I = gu.size(-1) / 2;
  CHK(gu.size(-1) == 2 * I);
  auto shape = gu.sizes().vec();
  shape.back() = I;
  auto out = torch::empty(shape, gu.options());
  const long long n = out.numel();
  if (n == 0) return out;
#define RUN(V)                                                                                                      \
  hipLaunchKernelGGL((geglu_kernel<T, V>), dim3((n / V + 255) / 256), dim3(256), 0, cur_stream(), P<T>(gu), M<T>(out), n, I)
  BY_TYPE(dt, {
    if (I % 4 == 0) RUN(4);
    else RUN(1);
  });
#undef RUN
  return out;
}

// fp32 whatever the input is
Tensor soft_cap(Tensor x, double cap) {
  const auto dt = io_type(x);
  CHK(cap > 0);
  auto out = torch::empty(x.sizes(), x.options().dtype(torch::kFloat32));
  const long long n = x.numel();
  if (n == 0) return out;
#define RUN(V)                                                                                                   \
  hipLaunchKernelGGL((soft_cap_kernel<T, V>), dim3((n / V + 255) / 256), dim3(256), 0, cur_stream(), P<T>(x), M<float>(out), n, \
                     (float)cap)
  BY_TYPE(dt, {
    if (n % 4 == 0) RUN(4);
    else RUN(1);
  });
#undef RUN
  return out;
}

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.def("embed_pairs", &embed_pairs, "embeddings of tokens and of token pairs");
  m.def("depth_norm", &depth_norm, "stream + outputs joins the streams so far; their average, its norms and convolution");
  m.def("geglu_packed", &geglu_packed, "gelu_tanh(gate) * up on a packed projection, any width, bf16 or fp32");
  m.def("soft_cap", &soft_cap, "cap tanh(x / cap), fp32");
}
