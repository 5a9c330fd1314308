// Attention with rotary positions, causal or over a sliding window that keeps
// the first tokens in sight (mode KEPT of attn_rows.h), with one or two maps
// per head: what norms, turns, appends and copies rows, and the entry point.
//
// A cache holds the first `keep` positions in rows of their own and the others
// in a ring of the rows that are left. Causal prompts read the cache itself,
// windowed ones a workspace of what their window still needs of it (the first
// tokens, then the window's) and the chunk.

#include "attn_rows.h"

// columns and widths of the sources; qm, km: query and key heads times maps
struct TurnArgs { int qm, km, rot, kN, k_at, v_at, pairs, late; };

// Rows of the workspace before the chunk, out of the cache.
template <typename T>
__global__ __launch_bounds__(256) void kept_history_kernel(
    const T* __restrict__ kc, const T* __restrict__ vc, T* __restrict__ kw, T* __restrict__ vw,
    KVShape ring, KVShape ws, int G, int km, int keep, int kept_rows, int base, Step step) {
  const int row = blockIdx.x, b = blockIdx.y, slot = max(step.slot(b), 0);
  const int src = place_of(row < kept_rows ? row : base + row - kept_rows, keep, keep, ring.mod);
  typedef Layout<T> L;
  const int kdims = sizeof(T) == 2 ? ws.kc * 32 : ws.dim, vdims = sizeof(T) == 2 ? ws.vg * 16 : ws.vdim;
  for (int i = threadIdx.x; i < km * kdims; i += 256) {
    const int g = i / kdims, d = i - g * kdims;
    kw[L::kbase(ws, (size_t)b * km + g) + L::k(ws, row, d)] = kc[L::kbase(ring, (size_t)slot * km + g) + L::k(ring, src, d)];
  }
  for (int i = threadIdx.x; i < G * vdims; i += 256) {
    const int g = i / vdims, c = i - g * vdims;
    vw[L::vbase(ws, (size_t)b * G + g) + L::v(ws, row, c)] = vc[L::vbase(ring, (size_t)slot * G + g) + L::v(ring, src, c)];
  }
}

// One block per token, 16 lanes a head: an RMS norm before the rotation (where
// there are weights), the rotation, an RMS norm after it; q to the workspace
// [B,S,qm,qd], k and v into the cache (what later steps can see) and into the
// workspace at rows hist+s (where there is one). Blocks past S fill the
// workspace's last tile with zeros. kv null: only q.
template <typename T>
__global__ __launch_bounds__(256) void turn_append_kernel(
    const T* __restrict__ proj, const T* __restrict__ kv, const T* __restrict__ qn, const T* __restrict__ kn,
    const float* __restrict__ freq, T* __restrict__ qw, T* __restrict__ kc, T* __restrict__ vc, T* __restrict__ kw,
    T* __restrict__ vw, KVShape ring, KVShape ws, int hist, TurnArgs r, AttnArgs a, Step step) {
  __shared__ float heads[16][264], turn_cos[128], turn_sin[128];
  const int s = blockIdx.x, b = blockIdx.y;
  const int slot = step.slot(b), len = step.decode ? 1 : step.len(b, a.S);
  typedef Layout<T> L;
  const bool live = s < len && slot >= 0;
  const int dim = ring.dim, vdim = ring.vdim;
  const int kdims = sizeof(T) == 2 ? ws.kc * 32 : dim, vdims = sizeof(T) == 2 ? ws.vg * 16 : vdim;
  const size_t tok = (size_t)b * a.S + s;
  const int pos = live ? step.first(b) + s : 0, half = r.rot / 2;
  const int crow = place_of(pos, a.keep, a.keep, ring.mod);
  const bool stay = kv && live && (pos < a.keep || s >= len - ring.mod) && crow < ring.rows;
  for (int i = threadIdx.x; i < half; i += 256) sincosf((float)pos * freq[i], &turn_sin[i], &turn_cos[i]);
  __syncthreads();
  const int l16 = threadIdx.x & 15;
  float* head = heads[threadIdx.x >> 4];
  for (int i = threadIdx.x >> 4; i < r.qm + (kv ? r.km : 0); i += 16) {
    const bool is_q = i < r.qm;
    const int h = is_q ? i : i - r.qm;
    if (is_q && s >= a.S) continue;
    if (!is_q && !stay && !kw) continue;
    const T *src = is_q ? proj + tok * a.N + a.q_at + h * dim : kv + tok * r.kN + r.k_at + h * dim, *wt = is_q ? qn : kn;
    const bool vec = ((dim | (is_q ? a.q_at | a.N : r.k_at | r.kN)) & 7) == 0;
    float x[16], ss = 0.f;
#pragma unroll
    for (int p = 0; p < 2; ++p) {
      const int d = p * 128 + l16 * 8;
#pragma unroll
      for (int j = 0; j < 8; ++j) x[p * 8 + j] = 0.f;
      if (live && d < dim) {
        if (vec) { ld4(src + d, x + p * 8); ld4(src + d + 4, x + p * 8 + 4); }
        else
#pragma unroll
          for (int j = 0; j < 8; ++j)
            if (d + j < dim) x[p * 8 + j] = ld(src + d + j);
      }
#pragma unroll
      for (int j = 0; j < 8; ++j) ss += x[p * 8 + j] * x[p * 8 + j];
    }
    if (wt) {
      const float inv = 1.f / sqrtf(row_sum(ss) / (float)dim + a.eps);
#pragma unroll
      for (int p = 0; p < 2; ++p)
#pragma unroll
        for (int j = 0; j < 8; ++j) {
          const int d = p * 128 + l16 * 8 + j;
          if (d < dim) x[p * 8 + j] *= inv * ld(wt + d);
        }
    }
#pragma unroll
    for (int p = 0; p < 2; ++p)
      if (p * 128 + l16 * 8 < r.rot) {
        st4(head + p * 128 + l16 * 8, x + p * 8);
        st4(head + p * 128 + l16 * 8 + 4, x + p * 8 + 4);
      }
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");  // a head's lanes are of one wave
    ss = 0.f;
#pragma unroll
    for (int p = 0; p < 2; ++p)
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        const int d = p * 128 + l16 * 8 + j;
        if (d < r.rot) {
          const bool second = r.pairs ? d & 1 : d >= half;
          const int n = r.pairs ? d >> 1 : second ? d - half : d;
          const float other = head[r.pairs ? d ^ 1 : second ? n : d + half];
          x[p * 8 + j] = x[p * 8 + j] * turn_cos[n] + (second ? other : -other) * turn_sin[n];
        }
        ss += x[p * 8 + j] * x[p * 8 + j];
      }
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
    if (r.late) {
      const float inv = 1.f / sqrtf(row_sum(ss) / (float)dim + a.eps);
#pragma unroll
      for (int j = 0; j < 16; ++j) x[j] *= inv;
    }
#pragma unroll
    for (int p = 0; p < 2; ++p) {
      const int d = p * 128 + l16 * 8, width = is_q ? a.qd : kdims;
      if (d >= width) continue;
      T* dst[2] = {nullptr, nullptr};
      if (is_q) dst[0] = qw + (tok * r.qm + h) * a.qd + d;
      else {
        if (stay) dst[0] = kc + L::kbase(ring, (size_t)slot * r.km + h) + L::k(ring, crow, d);
        if (kw) dst[1] = kw + L::kbase(ws, (size_t)b * r.km + h) + L::k(ws, hist + s, d);
      }
#pragma unroll
      for (int o = 0; o < 2; ++o)
        if (dst[o]) {
          if (sizeof(T) == 2 || (dim & 7) == 0) { st4(dst[o], x + p * 8); st4(dst[o] + 4, x + p * 8 + 4); }
          else
#pragma unroll
            for (int j = 0; j < 8; ++j)
              if (d + j < width) st(dst[o] + j, x[p * 8 + j]);
        }
    }
  }
  if (!kv || (!stay && !vw)) return;
  for (int i = threadIdx.x; i < a.G * vdims; i += 256) {
    const int g = i / vdims, c = i - g * vdims;
    const float f = live && c < vdim ? ld(kv + tok * r.kN + r.v_at + g * vdim + c) : 0.f;
    if (stay) st(vc + L::vbase(ring, (size_t)slot * a.G + g) + L::v(ring, crow, c), f);
    if (vw) st(vw + L::vbase(ws, (size_t)b * a.G + g) + L::v(ws, hist + s, c), f);
  }
}

// ===========================================================================
// host side
// ===========================================================================

// q: H * maps heads of proj from q_at on; keys and values: columns of kv, or
// already in the cache (kv null). window 0: causal.
void rotary_attn(Tensor proj, int64_t q_at, OptT kv, int64_t k_at, int64_t v_at, int64_t H, int64_t G, int64_t dim,
                 int64_t vdim, int64_t maps, double scale, double cap, int64_t window, int64_t keep, bool pairs,
                 bool late_norm, double eps, double gain, OptT q_norm, OptT k_norm, Tensor freq, OptT lam, Tensor kc,
                 Tensor vc, OptT slots, OptT positions, OptT lens, int64_t start, bool decode, Tensor out, int64_t out_at,
                 double out_scale) {
  const auto dt = io_type(proj);
  const bool bf = dt == torch::kBFloat16, windowed = window > 0;
  CHK(proj.dim() == 3 && out.dim() == 3 && out.size(0) == proj.size(0) && out.size(1) == proj.size(1));
  for (const Tensor& t : {kc, vc, out}) check_io(t, dt);
  check_io(freq, torch::kFloat32);
  const int B = proj.size(0), S = proj.size(1), N = proj.size(2), rot = 2 * freq.numel();
  CHK(H > 0 && G > 0 && H % G == 0 && dim > 0 && vdim > 0 && dim <= 256 && vdim <= 256 && (maps == 1 || maps == 2));
  CHK(rot <= dim && window >= 0 && window < INT_MAX && keep >= 0 && keep < INT_MAX / 2 && (windowed || keep == 0));
  CHK(q_at >= 0 && q_at + H * maps * dim <= N && out_at + H * vdim <= out.size(2) && out_at % 4 == 0 && out.size(2) % 4 == 0);
  CHK((!decode || S == 1) && (maps == 1 || lam) && (kv || !windowed));
  for (const OptT& t : {q_norm, k_norm})
    if (t) { check_io(*t, dt); CHK(t->numel() == dim); }
  if (lam) { check_io(*lam, torch::kFloat32); CHK(lam->numel() == 1); }
  if (kv) {
    check_io(*kv, dt);
    CHK(kv->dim() == 3 && kv->size(0) == B && kv->size(1) == S && k_at >= 0 && v_at >= 0);
    CHK(k_at + G * maps * dim <= kv->size(2) && v_at + G * vdim <= kv->size(2));
  }
  if (B == 0 || S == 0) return;
  KVShape ring = cache_shape(bf, G, dim, vdim, kc, vc, maps);
  CHK(slots || B <= kc.size(0));
  // a cache of fewer rows holds sequences that end before
  CHK(decode || (windowed && keep + window <= ring.rows) || start + S <= ring.rows);
  ring.mod = std::max<int>(1, ring.rows - (int)keep);
  const Step step = make_step(slots, positions, lens, start, decode, B);
  const AttnArgs a{S, (int)H, (int)G, N, (int)out.size(2), (int)q_at, 0, 0, 0, (int)out_at,
                   bf ? ring.kc * 32 : (int)dim, (float)scale, (float)eps, (float)out_scale,
                   windowed ? (int)window : INT_MAX, 0, (int)keep, !windowed, (float)cap, (float)gain,
                   lam ? lam->data_ptr<float>() : nullptr};
  const TurnArgs r{(int)(H * maps), (int)(G * maps), rot, kv ? (int)kv->size(2) : 0, (int)k_at, (int)v_at, pairs, late_norm};
  auto qw = torch::empty({B, S, H * maps, a.qd}, proj.options());
  const hipStream_t stream = cur_stream();
  auto append = [&](int blocks, const KVShape& ws, Tensor* wk, Tensor* wv, int hist) {
    BY_TYPE(dt, {
      hipLaunchKernelGGL((turn_append_kernel<T>), dim3(blocks, B), dim3(256), 0, stream, P<T>(proj),
                         kv ? P<T>(*kv) : nullptr, q_norm ? P<T>(*q_norm) : nullptr, k_norm ? P<T>(*k_norm) : nullptr,
                         freq.data_ptr<float>(), M<T>(qw), M<T>(kc), M<T>(vc), wk ? M<T>(*wk) : nullptr,
                         wv ? M<T>(*wv) : nullptr, ring, ws, hist, r, a, step);
    });
  };
  if (decode) {
    append(1, ring, nullptr, nullptr, 0);
    if (maps == 2) decode_rows<KEPT, 2>(bf, B, qw, kc, vc, nullptr, nullptr, nullptr, nullptr, 0, out, ring, (int)keep, a, step);
    else decode_rows<KEPT>(bf, B, qw, kc, vc, nullptr, nullptr, nullptr, nullptr, 0, out, ring, (int)keep, a, step);
    return;
  }
  if (!windowed) {
    append(S, ring, nullptr, nullptr, 0);
    if (maps == 2) prefill_rows<KEPT, 2>(bf, B, qw, kc, vc, nullptr, nullptr, nullptr, nullptr, out, ring, (int)start, 0, a, step);
    else prefill_rows<KEPT>(bf, B, qw, kc, vc, nullptr, nullptr, nullptr, nullptr, out, ring, (int)start, 0, a, step);
    return;
  }
  // the first tokens that lie before the window, then the window's, then the chunk
  const int base = (int)std::max<int64_t>(0, start - (window - 1)), kept_rows = std::min((int)keep, base);
  const int hist = kept_rows + (int)start - base;
  Workspace w(bf, ring, proj, B, G, hist, S, maps);
  BY_TYPE(dt, {
    if (hist > 0)
      hipLaunchKernelGGL((kept_history_kernel<T>), dim3(hist, B), dim3(256), 0, stream, P<T>(kc), P<T>(vc), M<T>(w.k),
                         M<T>(w.v), ring, w.shape, (int)G, r.km, (int)keep, kept_rows, base, step);
  });
  append(w.fill, w.shape, &w.k, &w.v, hist);
  const int from = std::max((int)keep, base);
  if (maps == 2) prefill_rows<KEPT, 2>(bf, B, qw, w.k, w.v, nullptr, nullptr, nullptr, nullptr, out, w.shape, hist, from, a, step);
  else prefill_rows<KEPT>(bf, B, qw, w.k, w.v, nullptr, nullptr, nullptr, nullptr, out, w.shape, hist, from, a, step);
}

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.def("rotary_attn", &rotary_attn, "rotary attention: causal or windowed with kept first tokens, one or two maps");
}
