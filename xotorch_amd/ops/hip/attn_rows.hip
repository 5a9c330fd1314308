// Attention over a window of the sequence with a bias per distance, and within
// chunks of it (modes WINDOW and CHUNK of attn_rows.h): what norms, appends and
// copies rows, and the entry points. Norms are over whole projections (WINDOW)
// or per head (CHUNK, whose values may be mixed with an earlier layer's).

#include "attn_rows.h"

// Keys of the window before a chunk, ring -> workspace rows [0, hist).
template <typename T>
__global__ __launch_bounds__(256) void window_history_kernel(
    const T* __restrict__ kc, const T* __restrict__ vc, T* __restrict__ kw, T* __restrict__ vw,
    KVShape ring, KVShape ws, int G, int base, int hist, Step step) {
  const int row = blockIdx.x, g = blockIdx.y, b = blockIdx.z;
  const int slot = step.slot(b);
  const int src = (base + row) % ring.mod;
  typedef Layout<T> L;
  const size_t kr = L::kbase(ring, (size_t)max(slot, 0) * G + g), vr = L::vbase(ring, (size_t)max(slot, 0) * G + g);
  const size_t kd = L::kbase(ws, (size_t)b * G + g), vd = L::vbase(ws, (size_t)b * G + g);
  const int kdims = sizeof(T) == 2 ? ws.kc * 32 : ws.dim, vdims = sizeof(T) == 2 ? ws.vg * 16 : ws.vdim;
  for (int d = threadIdx.x; d < kdims + vdims; d += 256) {
    if (d < kdims) kw[kd + L::k(ws, row, d)] = slot < 0 ? (T)0 : kc[kr + L::k(ring, src, d)];
    else vw[vd + L::v(ws, row, d - kdims)] = slot < 0 ? (T)0 : vc[vr + L::v(ring, src, d - kdims)];
  }
}

// One block per token: RMS norm over the whole q and k projections, q to the
// workspace [B,S,H,qd] (zero-padded dims), k and v into the ring (the last
// ring.rows tokens of the chunk) and, in prefill, into the workspace at rows
// hist+s. Blocks past S fill the workspace's last tile with zeros.
template <typename T>
__global__ __launch_bounds__(256) void qk_norm_append_kernel(
    const T* __restrict__ proj, const T* __restrict__ qn, const T* __restrict__ kn, T* __restrict__ qw,
    T* __restrict__ kc, T* __restrict__ vc, T* __restrict__ kw, T* __restrict__ vw,
    KVShape ring, KVShape ws, int hist, AttnArgs a, Step step) {
  const int s = blockIdx.x, b = blockIdx.y;
  const int slot = step.slot(b), len = step.decode ? 1 : step.len(b, a.S);
  typedef Layout<T> L;
  const bool live = s < len && slot >= 0;
  const int kdims = sizeof(T) == 2 ? ws.kc * 32 : ws.dim, vdims = sizeof(T) == 2 ? ws.vg * 16 : ws.vdim;
  if (!live) {
    if (s < a.S)
      for (int i = threadIdx.x; i < a.H * a.qd; i += 256) st(qw + ((size_t)b * a.S + s) * a.H * a.qd + i, 0.f);
    if (kw)
      for (int g = 0; g < a.G; ++g) {
        const size_t kd = L::kbase(ws, (size_t)b * a.G + g), vd = L::vbase(ws, (size_t)b * a.G + g);
        for (int d = threadIdx.x; d < kdims + vdims; d += 256) {
          if (d < kdims) st(kw + kd + L::k(ws, hist + s, d), 0.f);
          else st(vw + vd + L::v(ws, hist + s, d - kdims), 0.f);
        }
      }
    return;
  }
  const T* row = proj + ((size_t)b * a.S + s) * a.N;
  __shared__ float red[8];
  const int dim = ring.dim, nq = a.H * dim, nk = a.G * dim;
  const bool vec = ((dim | a.q_at | a.k_at | a.N) & 7) == 0;
  float qs = 0.f, ks = 0.f;
  if (vec) {
    for (int i = threadIdx.x * 4; i < nq + nk; i += 1024) {
      float x[4];
      ld4(row + (i < nq ? a.q_at + i : a.k_at + i - nq), x);
      const float f = x[0] * x[0] + x[1] * x[1] + x[2] * x[2] + x[3] * x[3];
      if (i < nq) qs += f;
      else ks += f;
    }
  } else {
    for (int i = threadIdx.x; i < nq; i += 256) { const float f = ld(row + a.q_at + i); qs += f * f; }
    for (int i = threadIdx.x; i < nk; i += 256) { const float f = ld(row + a.k_at + i); ks += f * f; }
  }
  const float qi = 1.f / sqrtf(block_sum(qs, red) / (float)nq + a.eps);
  const float ki = 1.f / sqrtf(block_sum(ks, red + 4) / (float)nk + a.eps);
  T* qrow = qw + ((size_t)b * a.S + s) * a.H * a.qd;
  const int pos = step.first(b) + s;
  const bool keep = s >= len - ring.rows;
  const int rrow = pos % ring.rows;
  if (vec) {
    // 8 channels at a time: they lie side by side in q rows and in both key
    // layouts; padded channels are zero
    const int gq = a.qd >> 3, gk = kdims >> 3;
    for (int i = threadIdx.x; i < a.H * gq + a.G * gk; i += 256) {
      const bool is_q = i < a.H * gq;
      const int e = is_q ? i : i - a.H * gq, h = e / (is_q ? gq : gk), d = (e - h * (is_q ? gq : gk)) * 8;
      float x[8], w[8];
#pragma unroll
      for (int j = 0; j < 8; ++j) x[j] = 0.f;
      if (d < dim) {
        const T *src = row + (is_q ? a.q_at : a.k_at) + h * dim + d, *wt = (is_q ? qn : kn) + h * dim + d;
        ld4(src, x);
        ld4(src + 4, x + 4);
        ld4(wt, w);
        ld4(wt + 4, w + 4);
#pragma unroll
        for (int j = 0; j < 8; ++j) x[j] *= (is_q ? qi : ki) * w[j];
      }
      if (is_q) {
        st4(qrow + h * a.qd + d, x);
        st4(qrow + h * a.qd + d + 4, x + 4);
        continue;
      }
      if (keep) {
        T* dst = kc + L::kbase(ring, (size_t)slot * a.G + h) + L::k(ring, rrow, d);
        st4(dst, x);
        st4(dst + 4, x + 4);
      }
      if (kw) {
        T* dst = kw + L::kbase(ws, (size_t)b * a.G + h) + L::k(ws, hist + s, d);
        st4(dst, x);
        st4(dst + 4, x + 4);
      }
    }
  } else {
    for (int i = threadIdx.x; i < a.H * a.qd; i += 256) {
      const int h = i / a.qd, d = i - h * a.qd, j = h * dim + d;
      st(qrow + i, d < dim ? ld(row + a.q_at + j) * qi * ld(qn + j) : 0.f);
    }
    for (int i = threadIdx.x; i < a.G * kdims; i += 256) {
      const int g = i / kdims, d = i - g * kdims, j = g * dim + d;
      const float f = d < dim ? ld(row + a.k_at + j) * ki * ld(kn + j) : 0.f;
      if (keep) st(kc + L::kbase(ring, (size_t)slot * a.G + g) + L::k(ring, rrow, d), f);
      if (kw) st(kw + L::kbase(ws, (size_t)b * a.G + g) + L::k(ws, hist + s, d), f);
    }
  }
  for (int i = threadIdx.x; i < a.G * vdims; i += 256) {
    const int g = i / vdims, c = i - g * vdims;
    const float f = c < ring.vdim ? ld(row + a.v_at + g * ring.vdim + c) : 0.f;
    if (keep) st(vc + L::vbase(ring, (size_t)slot * a.G + g) + L::v(ring, rrow, c), f);
    if (kw) st(vw + L::vbase(ws, (size_t)b * a.G + g) + L::v(ws, hist + s, c), f);
  }
}

// Values of an earlier layer for the same tokens, mixed in before caching.
struct ValueMix {
  const void *first, *lambda;
  long long row_stride, tok_stride;
};

// One block per token: an RMS norm per head on q and k (16 lanes a head), q to
// the workspace, k and the mixed v into the cache (tokens of the last chunk of
// the sequence only) and, in prefill, into the workspace at rows hist+s. Blocks
// past S fill the workspace's last tile with zeros.
template <typename T>
__global__ __launch_bounds__(256) void head_norm_append_kernel(
    const T* __restrict__ proj, const T* __restrict__ qn, const T* __restrict__ kn, ValueMix mix, T* __restrict__ qw,
    T* __restrict__ kc, T* __restrict__ vc, T* __restrict__ kw, T* __restrict__ vw,
    KVShape ring, KVShape ws, int hist, AttnArgs a, Step step) {
  const int s = blockIdx.x, b = blockIdx.y;
  const int slot = step.slot(b), len = step.decode ? 1 : step.len(b, a.S);
  typedef Layout<T> L;
  const bool live = s < len && slot >= 0;
  const int dim = ring.dim, vdim = ring.vdim;
  const int kdims = sizeof(T) == 2 ? ws.kc * 32 : dim, vdims = sizeof(T) == 2 ? ws.vg * 16 : vdim;
  const size_t tok = (size_t)b * a.S + s;
  const T* row = proj + tok * a.N;
  const int pos = live ? step.first(b) + s : 0;
  // the chunk of the row's last token is what later steps read
  const int last = live ? step.first(b) + len - 1 : 0, crow = pos % ring.mod;
  const bool keep = live && pos >= last - last % ring.mod && crow < ring.rows;
  const int l16 = threadIdx.x & 15;
  const bool vec = ((dim | a.q_at | a.k_at | a.N) & 7) == 0;
  for (int i = threadIdx.x >> 4; i < a.H + a.G; i += 16) {
    const bool is_q = i < a.H;
    const int h = is_q ? i : i - a.H;
    if (is_q && s >= a.S) continue;
    if (!is_q && !keep && !kw) continue;
    const T *src = row + (is_q ? a.q_at : a.k_at) + h * dim, *wt = is_q ? qn : kn;
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
#pragma unroll
        for (int j = 0; j < 8; ++j) ss += x[p * 8 + j] * x[p * 8 + j];
      }
    }
    const float inv = 1.f / sqrtf(row_sum(ss) / (float)dim + a.eps);
#pragma unroll
    for (int p = 0; p < 2; ++p) {
      const int d = p * 128 + l16 * 8, width = is_q ? a.qd : kdims;
      if (d >= width) continue;
#pragma unroll
      for (int j = 0; j < 8; ++j) x[p * 8 + j] *= d + j < dim ? inv * ld(wt + d + j) : 0.f;
      T* dst[2] = {nullptr, nullptr};
      if (is_q) dst[0] = qw + (tok * a.H + h) * a.qd + d;
      else {
        if (keep) dst[0] = kc + L::kbase(ring, (size_t)slot * a.G + h) + L::k(ring, crow, d);
        if (kw) dst[1] = kw + L::kbase(ws, (size_t)b * a.G + h) + L::k(ws, hist + s, d);
      }
#pragma unroll
      for (int o = 0; o < 2; ++o)
        if (dst[o]) {
          if (sizeof(T) == 2 || vec) { st4(dst[o], x + p * 8); st4(dst[o] + 4, x + p * 8 + 4); }
          else
#pragma unroll
            for (int j = 0; j < 8; ++j)
              if (d + j < width) st(dst[o] + j, x[p * 8 + j]);
        }
    }
  }
  if (!keep && !vw) return;
  const float lam = mix.first ? ld((const T*)mix.lambda) : 0.f;
  for (int i = threadIdx.x; i < a.G * vdims; i += 256) {
    const int g = i / vdims, c = i - g * vdims;
    float f = 0.f;
    if (live && c < vdim) {
      f = ld(row + a.v_at + g * vdim + c);
      if (mix.first)
        f = (1.f - lam) * f + lam * ld((const T*)mix.first + b * mix.row_stride + s * mix.tok_stride + g * vdim + c);
    }
    if (keep) st(vc + L::vbase(ring, (size_t)slot * a.G + g) + L::v(ring, crow, c), f);
    if (vw) st(vw + L::vbase(ws, (size_t)b * a.G + g) + L::v(ws, hist + s, c), f);
  }
}

// ===========================================================================
// host side
// ===========================================================================

void window_attn(Tensor proj, int64_t q_at, int64_t k_at, int64_t v_at, int64_t g_at, int64_t H, int64_t G,
                 int64_t dim, int64_t vdim, Tensor q_norm, Tensor k_norm, Tensor bucket, Tensor rel, double scale,
                 double eps, int64_t window, Tensor kc, Tensor vc, OptT slots, OptT positions, OptT lens,
                 int64_t start, bool decode, Tensor out, int64_t out_at, double out_scale) {
  const auto dt = io_type(proj);
  const bool bf = dt == torch::kBFloat16;
  CHK(proj.dim() == 3 && out.dim() == 3 && out.size(0) == proj.size(0) && out.size(1) == proj.size(1));
  for (const Tensor& t : {q_norm, k_norm, rel, kc, vc, out}) check_io(t, dt);
  check_io(bucket, torch::kInt32);
  const int B = proj.size(0), S = proj.size(1), N = proj.size(2);
  CHK(H > 0 && G > 0 && H % G == 0 && dim > 0 && vdim > 0 && dim <= 256 && vdim <= 256 && window > 0);
  CHK(q_at + H * dim <= N && k_at + G * dim <= N && v_at + G * vdim <= N && g_at + H <= N);
  CHK(out_at + H * vdim <= out.size(2) && out_at % 4 == 0 && out.size(2) % 4 == 0);
  CHK(q_norm.numel() == H * dim && k_norm.numel() == G * dim && rel.dim() == 2 && rel.size(1) == H);
  CHK(bucket.numel() > 0 && (!decode || S == 1));
  if (B == 0 || S == 0) return;
  const KVShape ring = cache_shape(bf, G, dim, vdim, kc, vc);
  CHK(slots || B <= kc.size(0));
  const Step step = make_step(slots, positions, lens, start, decode, B);
  const AttnArgs a{S, (int)H, (int)G, N, (int)out.size(2), (int)q_at, (int)k_at, (int)v_at, (int)g_at, (int)out_at,
                   bf ? ring.kc * 32 : (int)dim, (float)scale, (float)eps, (float)out_scale, (int)window,
                   (int)bucket.numel()};
  auto qw = torch::empty({B, S, H, a.qd}, proj.options());
  const hipStream_t stream = cur_stream();
  const int* bk = bucket.data_ptr<int>();
  const int rel_rows = rel.size(0);
  if (decode) {
    BY_TYPE(dt, {
      hipLaunchKernelGGL((qk_norm_append_kernel<T>), dim3(1, B), dim3(256), 0, stream, P<T>(proj), P<T>(q_norm),
                         P<T>(k_norm), M<T>(qw), M<T>(kc), M<T>(vc), (T*)nullptr, (T*)nullptr, ring, ring, 0, a, step);
    });
    decode_rows<WINDOW>(bf, B, qw, kc, vc, proj.data_ptr(), nullptr, bk, rel.data_ptr(), rel_rows, out, ring, 0, a, step);
    return;
  }
  // the workspace: what the window still holds of earlier chunks, then this chunk
  const int base = (int)std::max<int64_t>(0, start - (window - 1)), hist = (int)start - base;
  CHK(hist <= ring.rows);
  Workspace w(bf, ring, proj, B, G, hist, S);
  BY_TYPE(dt, {
    if (hist > 0)
      hipLaunchKernelGGL((window_history_kernel<T>), dim3(hist, G, B), dim3(256), 0, stream, P<T>(kc), P<T>(vc),
                         M<T>(w.k), M<T>(w.v), ring, w.shape, (int)G, base, hist, step);
    hipLaunchKernelGGL((qk_norm_append_kernel<T>), dim3(w.fill, B), dim3(256), 0, stream, P<T>(proj), P<T>(q_norm),
                       P<T>(k_norm), M<T>(qw), M<T>(kc), M<T>(vc), M<T>(w.k), M<T>(w.v), ring, w.shape, hist, a, step);
  });
  prefill_rows<WINDOW>(bf, B, qw, w.k, w.v, proj.data_ptr(), nullptr, bk, rel.data_ptr(), out, w.shape, hist, base, a,
                       step);
}

void chunk_attn(Tensor proj, int64_t q_at, int64_t k_at, int64_t v_at, int64_t H, int64_t G, int64_t dim, int64_t vdim,
                Tensor q_norm, Tensor k_norm, Tensor sinks, OptT first, OptT lambda, double scale, double eps,
                int64_t chunk, Tensor kc, Tensor vc, OptT slots, OptT positions, OptT lens, int64_t start, bool decode,
                Tensor out, int64_t out_at, double out_scale) {
  const auto dt = io_type(proj);
  const bool bf = dt == torch::kBFloat16;
  CHK(proj.dim() == 3 && out.dim() == 3 && out.size(0) == proj.size(0) && out.size(1) == proj.size(1));
  for (const Tensor& t : {q_norm, k_norm, sinks, kc, vc, out}) check_io(t, dt);
  const int B = proj.size(0), S = proj.size(1), N = proj.size(2);
  CHK(H > 0 && G > 0 && H % G == 0 && dim > 0 && vdim > 0 && dim <= 256 && vdim <= 256 && chunk > 0);
  CHK(q_at + H * dim <= N && k_at + G * dim <= N && v_at + G * vdim <= N);
  CHK(out_at + H * vdim <= out.size(2) && out_at % 4 == 0 && out.size(2) % 4 == 0);
  CHK(q_norm.numel() == dim && k_norm.numel() == dim && sinks.numel() == H && (!decode || S == 1));
  if (B == 0 || S == 0) return;
  KVShape ring = cache_shape(bf, G, dim, vdim, kc, vc);
  CHK(slots || B <= kc.size(0));
  ring.mod = (int)std::min<int64_t>(chunk, INT_MAX);
  // positions within a chunk have rows of their own; a cache of fewer rows
  // holds sequences that end before
  CHK(decode || chunk <= ring.rows || start + S <= ring.rows);
  ValueMix mix{nullptr, nullptr, 0, 0};
  if (first) {
    CHK(lambda && lambda->numel() == 1);
    check_io(*lambda, dt);
    CHK(first->is_cuda() && first->scalar_type() == dt && first->dim() == 3 && first->size(0) == B &&
        first->size(1) == S && first->size(2) == G * vdim && first->stride(2) == 1);
    mix = ValueMix{first->data_ptr(), lambda->data_ptr(), (long long)first->stride(0), (long long)first->stride(1)};
  }
  const Step step = make_step(slots, positions, lens, start, decode, B);
  const AttnArgs a{S, (int)H, (int)G, N, (int)out.size(2), (int)q_at, (int)k_at, (int)v_at, 0, (int)out_at,
                   bf ? ring.kc * 32 : (int)dim, (float)scale, (float)eps, (float)out_scale, ring.mod, 0};
  auto qw = torch::empty({B, S, H, a.qd}, proj.options());
  const hipStream_t stream = cur_stream();
  if (decode) {
    BY_TYPE(dt, {
      hipLaunchKernelGGL((head_norm_append_kernel<T>), dim3(1, B), dim3(256), 0, stream, P<T>(proj), P<T>(q_norm),
                         P<T>(k_norm), mix, M<T>(qw), M<T>(kc), M<T>(vc), (T*)nullptr, (T*)nullptr, ring, ring, 0, a,
                         step);
    });
    decode_rows<CHUNK>(bf, B, qw, kc, vc, nullptr, sinks.data_ptr(), nullptr, nullptr, 0, out, ring, 0, a, step);
    return;
  }
  // the workspace begins with the chunk that `start` lies in
  const int hist = (int)(start % ring.mod), base = (int)start - hist;
  CHK(hist <= ring.rows);
  Workspace w(bf, ring, proj, B, G, hist, S);
  BY_TYPE(dt, {
    if (hist > 0)
      hipLaunchKernelGGL((window_history_kernel<T>), dim3(hist, G, B), dim3(256), 0, stream, P<T>(kc), P<T>(vc),
                         M<T>(w.k), M<T>(w.v), ring, w.shape, (int)G, base, hist, step);
    hipLaunchKernelGGL((head_norm_append_kernel<T>), dim3(w.fill, B), dim3(256), 0, stream, P<T>(proj), P<T>(q_norm),
                       P<T>(k_norm), mix, M<T>(qw), M<T>(kc), M<T>(vc), M<T>(w.k), M<T>(w.v), ring, w.shape, hist, a,
                       step);
  });
  prefill_rows<CHUNK>(bf, B, qw, w.k, w.v, nullptr, sinks.data_ptr(), nullptr, nullptr, out, w.shape, hist, base, a, step);
}

// Causal attention of prompt rows over workspaces in this file's layouts: q
// [B,S,H,qd], k and v of every head for positions [0, rows), rows >= start+S.
// sinks [H]; gates [B,S,N], of which columns g_at.. multiply the outputs.
void causal_attn(Tensor q, Tensor k, Tensor v, int64_t dim, int64_t vdim, int64_t rows, double scale, OptT slots,
                 OptT lens, int64_t start, Tensor out, int64_t out_at, double out_scale, OptT sinks, OptT gates,
                 int64_t g_at) {
  const auto dt = io_type(q);
  const bool bf = dt == torch::kBFloat16;
  for (const Tensor& t : {k, v, out}) check_io(t, dt);
  CHK(q.dim() == 4 && out.dim() == 3 && out.size(0) == q.size(0) && out.size(1) == q.size(1));
  const int B = q.size(0), S = q.size(1), H = q.size(2);
  KVShape ws{(int)dim, (int)vdim, (int)(dim + 31) / 32, (int)(vdim + 15) / 16, (int)rows, INT_MAX};
  CHK(dim > 0 && vdim > 0 && dim <= 256 && vdim <= 256 && rows >= start + S && (!bf || rows % 32 == 0));
  CHK(q.size(3) == (bf ? ws.kc * 32 : dim));
  CHK(k.numel() == (int64_t)B * H * rows * (bf ? ws.kc * 32 : dim));
  CHK(v.numel() == (int64_t)B * H * rows * (bf ? ws.vg * 16 : vdim));
  CHK(out_at + H * vdim <= out.size(2) && out_at % 4 == 0 && out.size(2) % 4 == 0);
  if (sinks) { check_io(*sinks, dt); CHK(sinks->numel() == H); }
  if (gates) {
    check_io(*gates, dt);
    CHK(gates->dim() == 3 && gates->size(0) == B && gates->size(1) == S && g_at >= 0 && g_at + H * vdim <= gates->size(2));
  }
  if (B == 0 || S == 0) return;
  const Step step = make_step(slots, c10::nullopt, lens, start, false, B);
  const AttnArgs a{S, H, H, gates ? (int)gates->size(2) : 0, (int)out.size(2), 0, 0, 0, (int)g_at, (int)out_at,
                   (int)q.size(3), (float)scale, 0.f, (float)out_scale, 0, 0};
  prefill_rows<CAUSAL>(bf, B, q, k, v, gates ? gates->data_ptr() : nullptr, sinks ? sinks->data_ptr() : nullptr, nullptr,
                       nullptr, out, ws, (int)start, 0, a, step);
}

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.def("window_attn", &window_attn, "sliding-window attention with distance bias, sink and head gates");
  m.def("chunk_attn", &chunk_attn, "attention within chunks of the sequence: linear distance bias, learned sinks, mixed values");
  m.def("causal_attn", &causal_attn, "causal attention of prompt rows over packed workspaces, sinks, gates",
        py::arg("q"), py::arg("k"), py::arg("v"), py::arg("dim"), py::arg("vdim"), py::arg("rows"), py::arg("scale"),
        py::arg("slots"), py::arg("lens"), py::arg("start"), py::arg("out"), py::arg("out_at"), py::arg("out_scale"),
        py::arg("sinks") = py::none(), py::arg("gates") = py::none(), py::arg("g_at") = 0);
}
