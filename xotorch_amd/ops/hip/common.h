// Shared by the token-mixer translation units: element access for bf16 and fp32,
// wave and block reductions, step rows, cache layouts, host-side checks.
#pragma once

#include <torch/extension.h>
#include <c10/hip/HIPStream.h>
#include <hip/hip_runtime.h>
#include <hip/hip_bf16.h>

#include <algorithm>
#include <climits>
#include <type_traits>

typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8;
typedef __attribute__((ext_vector_type(4))) float floatx4;
typedef __attribute__((ext_vector_type(4))) unsigned short ushort4_t;
typedef unsigned short bf16_t;

#define DEVINL __device__ __forceinline__

DEVINL float ld(const bf16_t* p) {
  union { float f; unsigned int i; } v;
  v.i = ((unsigned int)*p) << 16;
  return v.f;
}
DEVINL float ld(const float* p) { return *p; }
DEVINL bf16_t f2b(float f) {
  __hip_bfloat16 h = __float2bfloat16(f);  // round to nearest even
  return *reinterpret_cast<bf16_t*>(&h);
}
DEVINL void st(bf16_t* p, float f) { *p = f2b(f); }
DEVINL void st(float* p, float f) { *p = f; }

DEVINL void ld4(const float* p, float* o) {
  const floatx4 v = *(const floatx4*)p;
#pragma unroll
  for (int i = 0; i < 4; ++i) o[i] = v[i];
}
DEVINL void ld4(const bf16_t* p, float* o) {
  const ushort4_t v = *(const ushort4_t*)p;
#pragma unroll
  for (int i = 0; i < 4; ++i) { bf16_t u = v[i]; o[i] = ld(&u); }
}
typedef __attribute__((ext_vector_type(2))) float floatx2;
typedef __attribute__((ext_vector_type(2))) unsigned short ushort2_t;
DEVINL void ld2(const float* p, float* o) {
  const floatx2 v = *(const floatx2*)p;
  o[0] = v[0];
  o[1] = v[1];
}
DEVINL void ld2(const bf16_t* p, float* o) {
  const ushort2_t v = *(const ushort2_t*)p;
  bf16_t a = v[0], b = v[1];
  o[0] = ld(&a);
  o[1] = ld(&b);
}
DEVINL void st2(float* p, const float* o) {
  floatx2 v;
  v[0] = o[0];
  v[1] = o[1];
  *(floatx2*)p = v;
}
DEVINL void st2(bf16_t* p, const float* o) {
  ushort2_t v;
  v[0] = f2b(o[0]);
  v[1] = f2b(o[1]);
  *(ushort2_t*)p = v;
}
DEVINL void st4(float* p, const float* o) {
  floatx4 v;
#pragma unroll
  for (int i = 0; i < 4; ++i) v[i] = o[i];
  *(floatx4*)p = v;
}
DEVINL void st4(bf16_t* p, const float* o) {
  ushort4_t v;
#pragma unroll
  for (int i = 0; i < 4; ++i) v[i] = f2b(o[i]);
  *(ushort4_t*)p = v;
}
template <int V, typename T>
DEVINL void ldv(const T* p, float* o) {
  if (V == 4) ld4(p, o);
  else
#pragma unroll
    for (int i = 0; i < V; ++i) o[i] = ld(p + i);
}
template <int V, typename T>
DEVINL void stv(T* p, const float* o) {
  if (V == 4) st4(p, o);
  else
#pragma unroll
    for (int i = 0; i < V; ++i) st(p + i, o[i]);
}

// hardware exp2/log2/rcp (about one ulp each)
DEVINL float sigmoidf(float x) { return __builtin_amdgcn_rcpf(1.f + __expf(-x)); }
DEVINL float siluf(float x) { return x * sigmoidf(x); }
// 0.5 z (1 + tanh(sqrt(2/pi) (z + 0.044715 z^3))) as z sigmoid(2 sqrt(2/pi) (..))
DEVINL float gelu_tanh(float z) { return z * sigmoidf(1.5957691216057308f * (z + 0.044715f * z * z * z)); }
// log1p(e) = log(u) e / (u - 1) with u = 1 + e as rounded: exact where e is tiny
DEVINL float softplusf(float x) {
  const float e = __expf(-fabsf(x)), u = 1.f + e;
  return fmaxf(x, 0.f) + (u == 1.f ? e : __logf(u) * e * __builtin_amdgcn_rcpf(u - 1.f));
}

// sum over the 16 lanes of a DPP row, in every lane (row_ror:8, 4, 2, 1)
DEVINL float row_sum(float v) {
  v += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x128, 0xf, 0xf, true));
  v += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x124, 0xf, 0xf, true));
  v += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x122, 0xf, 0xf, true));
  v += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x121, 0xf, 0xf, true));
  return v;
}
DEVINL float wave_sum(float v) {
  v = row_sum(v);
  v += __shfl_xor(v, 16);
  v += __shfl_xor(v, 32);
  return v;
}
// maximum and minimum over the 16 lanes of a DPP row, in every lane
DEVINL float row_max(float v) {
  v = fmaxf(v, __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x128, 0xf, 0xf, true)));
  v = fmaxf(v, __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x124, 0xf, 0xf, true)));
  v = fmaxf(v, __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x122, 0xf, 0xf, true)));
  return fmaxf(v, __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x121, 0xf, 0xf, true)));
}
DEVINL int row_min(int v) {
  v = min(v, __builtin_amdgcn_update_dpp(0, v, 0x128, 0xf, 0xf, true));
  v = min(v, __builtin_amdgcn_update_dpp(0, v, 0x124, 0xf, 0xf, true));
  v = min(v, __builtin_amdgcn_update_dpp(0, v, 0x122, 0xf, 0xf, true));
  return min(v, __builtin_amdgcn_update_dpp(0, v, 0x121, 0xf, 0xf, true));
}
// sum over a block of 256 threads; `red` holds 4 floats and is free again
// after the next barrier
DEVINL float block_sum(float v, float* red) {
  v = wave_sum(v);
  if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
  __syncthreads();
  return red[0] + red[1] + red[2] + red[3];
}

// operands of 16x16 matrix products in either element type (fp32 throughout)
template <typename T> struct Frag;
template <> struct Frag<bf16_t> {
  typedef bf16x8 V;
  static constexpr int K = 32, PER = 8;  // k of a step, elements of a lane
};
template <> struct Frag<float> {
  typedef floatx4 V;
  static constexpr int K = 16, PER = 4;
};
// D[16 rows of a][16 rows of b] += over one k step
DEVINL floatx4 mma(const bf16x8& a, const bf16x8& b, floatx4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0);
}
DEVINL floatx4 mma(const floatx4& a, const floatx4& b, floatx4 c) {
#pragma unroll
  for (int i = 0; i < 4; ++i) c = __builtin_amdgcn_mfma_f32_16x16x4f32(a[i], b[i], c, 0, 0, 0);
  return c;
}
// a lane's elements k.. of a row of n; WHOLE: n is a multiple of the step
template <typename T, bool WHOLE>
DEVINL typename Frag<T>::V ld_frag(const T* row, int k, int n) {
  typedef typename Frag<T>::V V;
  if (WHOLE) return *(const V*)(row + k);
  union { V v; T e[Frag<T>::PER]; } u;
#pragma unroll
  for (int i = 0; i < Frag<T>::PER; ++i) u.e[i] = k + i < n ? row[k + i] : (T)0;
  return u.v;
}

struct Step {
  const int* slots;      // null: row b is slot b
  const int* positions;  // decode only
  const int* lens;       // prefill only; null: every row brings S tokens
  int npos, start, decode;
  DEVINL int slot(int b) const { return slots ? slots[b] : b; }
  DEVINL int first(int b) const { return decode ? positions[npos > 1 ? b : 0] : start; }
  DEVINL int len(int b, int S) const { return lens ? min(lens[b], S) : S; }
};

// ---------------------------------------------------------------------------
// key/value layouts
//   bf16, fragment-packed per (slot, kv head):
//     K [rows/16][KC][64 lanes][8]: lane = (d%32)/8*16 + row%16
//     V [VG][rows/32][64 lanes][8]: lane = (row%16)/4*16 + c%16,
//       element = (row%32)/16*4 + row%4
//     Scores are computed transposed (keys x queries), so the lane that holds
//     a query's probabilities for keys {4g..4g+3, 16+4g..16+4g+3} feeds them
//     straight into the second MFMA; V's element order follows that.
//   fp32: plain rows.
// ---------------------------------------------------------------------------

// Position p lies in row p % mod of a cache (the window or chunk length; a
// cache of whole sequences never wraps).
struct KVShape { int dim, vdim, kc, vg, rows, mod; };

template <typename T> struct Layout;
template <> struct Layout<bf16_t> {
  static DEVINL size_t kbase(const KVShape& s, size_t head) { return head * (size_t)(s.rows >> 4) * s.kc * 512; }
  static DEVINL size_t vbase(const KVShape& s, size_t head) { return head * (size_t)s.vg * (s.rows >> 5) * 512; }
  static DEVINL size_t k(const KVShape& s, int row, int d) {
    return (((size_t)(row >> 4) * s.kc + (d >> 5)) * 64 + ((d & 31) >> 3) * 16 + (row & 15)) * 8 + (d & 7);
  }
  static DEVINL size_t v(const KVShape& s, int row, int c) {
    return (((size_t)(c >> 4) * (s.rows >> 5) + (row >> 5)) * 64 + ((row & 15) >> 2) * 16 + (c & 15)) * 8 +
           ((row & 31) >> 4) * 4 + (row & 3);
  }
};
template <> struct Layout<float> {
  static DEVINL size_t kbase(const KVShape& s, size_t head) { return head * s.rows * (size_t)s.dim; }
  static DEVINL size_t vbase(const KVShape& s, size_t head) { return head * s.rows * (size_t)s.vdim; }
  static DEVINL size_t k(const KVShape& s, int row, int d) { return (size_t)row * s.dim + d; }
  static DEVINL size_t v(const KVShape& s, int row, int c) { return (size_t)row * s.vdim + c; }
};

// ===========================================================================
// host side
// ===========================================================================

#define CHK(x) TORCH_CHECK(x, #x)
using torch::Tensor;
using OptT = c10::optional<Tensor>;

static inline hipStream_t cur_stream() { return (hipStream_t)c10::hip::getCurrentHIPStream().stream(); }

static void check_io(const Tensor& t, torch::ScalarType dt) {
  TORCH_CHECK(t.is_cuda() && t.is_contiguous() && t.scalar_type() == dt, "contiguous GPU tensor of type ",
              c10::toString(dt), " expected, got ", c10::toString(t.scalar_type()), t.sizes());
}
static torch::ScalarType io_type(const Tensor& t) {
  const auto dt = t.scalar_type();
  TORCH_CHECK(dt == torch::kBFloat16 || dt == torch::kFloat32, "bfloat16 or float32 expected");
  check_io(t, dt);
  return dt;
}
static Tensor f32(const Tensor& like, std::vector<int64_t> shape) {
  return torch::empty(shape, like.options().dtype(torch::kFloat32));
}

static Step make_step(const OptT& slots, const OptT& positions, const OptT& lens, int64_t start, bool decode, int B) {
  Step s{};
  if (slots) { check_io(*slots, torch::kInt32); CHK(slots->numel() == B); s.slots = slots->data_ptr<int>(); }
  if (lens && !decode) { check_io(*lens, torch::kInt32); CHK(lens->numel() == B); s.lens = lens->data_ptr<int>(); }
  if (decode) {
    TORCH_CHECK(positions, "a decode step needs positions");
    check_io(*positions, torch::kInt32);
    CHK(positions->numel() == 1 || positions->numel() == B);
    s.positions = positions->data_ptr<int>();
    s.npos = positions->numel();
  }
  CHK(start >= 0);
  s.start = (int)start;
  s.decode = decode;
  return s;
}

template <typename T> static const T* P(const Tensor& t) { return (const T*)t.data_ptr(); }
template <typename T> static T* M(Tensor& t) { return (T*)t.data_ptr(); }

#define BY_TYPE(dt, ...)                                              \
  if (dt == torch::kBFloat16) { typedef bf16_t T; __VA_ARGS__; }      \
  else { typedef float T; __VA_ARGS__; }

