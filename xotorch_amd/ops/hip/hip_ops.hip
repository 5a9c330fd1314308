// xotorch_amd CDNA4 (gfx950 / MI355X) kernels for the transformer hot path.
//
// These replace the ops the reference delegates to torchtune
// (reference call sites cited per kernel below):
//   - fused residual-add + RMSNorm      (llm_utils.py:465-476)
//   - fused RoPE rotate + KV-cache append, dual layout (general_mha.py:78-106)
//   - GQA attention, prefill AND decode, on matrix cores
//     (general_mha.py:211-226): flash-forward / flash-decoding with online
//     softmax, v_mfma_f32_16x16x32_bf16 for scores and PV, streaming an
//     MFMA-fragment-packed KV cache with coalesced 1 KB wave loads
//   - decode projections (qkv/o/gate_up/down/lm_head, general_mha.py:83-102,
//     llm_utils.py:491-500): weight-streaming split-K GEMMs on
//     v_mfma_f32_32x32x16_bf16 over prepacked weight fragments (non-temporal
//     loads; a grouped variant runs every MoE expert in one launch, and a
//     W8A8 e4m3 variant halves the stream) — auto-picked per shape against
//     TunableOp-tuned hipBLASLt at runtime
//   - SwiGLU activation                  (llm_utils.py:491-500)
//
// Design notes:
//   * wave = 64 lanes; all block sizes are multiples of 64
//   * bf16 is loaded vectorized (ushort8 = 16 B per lane); the big streamed
//     operands (weights, KV) are pre-shuffled ONCE into MFMA fragment order
//     so every hot-loop load is a coalesced wave-wide 1 KB stream
//     (fragment-shaped 16 B gathers measured TA-bound at ~2 TB/s vs 5.5)
//   * everything is launch-shape-static so the whole decode step can be
//     captured in a hipGraph (lengths come from device tensors)
//
// Prefill projections (compute-bound) stay on hipBLASLt through torch —
// plain library GEMMs per the MI355X build rules; measured ~1.6 PF there.

#include <torch/extension.h>
#include <c10/hip/HIPStream.h>
#include <hip/hip_runtime.h>
#include <hip/hip_bf16.h>

#include <vector>

typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8;
typedef __attribute__((ext_vector_type(16))) float floatx16;
typedef __attribute__((ext_vector_type(4))) float floatx4;

typedef __attribute__((ext_vector_type(8))) unsigned short ushort8;
typedef __attribute__((ext_vector_type(4))) unsigned short ushort4_t;

#define DEVINL __device__ __forceinline__

DEVINL float b2f(unsigned short u) {
  union { float f; unsigned int i; } v;
  v.i = ((unsigned int)u) << 16;
  return v.f;
}

DEVINL unsigned short f2b(float f) {
  __hip_bfloat16 h = __float2bfloat16(f);  // round-to-nearest-even
  return *reinterpret_cast<unsigned short*>(&h);
}

// ---------------------------------------------------------------------------
// RMSNorm (optionally fused with residual add)
// one workgroup per row; 256 threads; row cached in registers between the
// two passes (up to 8 chunks of 8 bf16 per thread -> D <= 16384)
// ---------------------------------------------------------------------------

template <bool RESIDUAL>
__global__ __launch_bounds__(256) void rmsnorm_kernel(
    const unsigned short* __restrict__ x, const unsigned short* __restrict__ res,
    const unsigned short* __restrict__ w, unsigned short* __restrict__ out,
    unsigned short* __restrict__ res_out, int D, float eps, float w_bias) {
  const int row = blockIdx.x;
  const size_t off = (size_t)row * D;
  float vals[64];
  float acc = 0.f;
#pragma unroll
  for (int c = 0; c < 8; ++c) {
    const int i = threadIdx.x * 8 + c * 256 * 8;
    if (i < D) {
      ushort8 v = *(const ushort8*)(x + off + i);
      if (RESIDUAL) {
        ushort8 r = *(const ushort8*)(res + off + i);
        ushort8 s;
#pragma unroll
        for (int j = 0; j < 8; ++j) {
          const float f = b2f(v[j]) + b2f(r[j]);
          vals[c * 8 + j] = f;
          s[j] = f2b(f);
          acc += f * f;
        }
        *(ushort8*)(res_out + off + i) = s;
      } else {
#pragma unroll
        for (int j = 0; j < 8; ++j) {
          const float f = b2f(v[j]);
          vals[c * 8 + j] = f;
          acc += f * f;
        }
      }
    }
  }
  // wave reduce then cross-wave through LDS
#pragma unroll
  for (int m = 32; m > 0; m >>= 1) acc += __shfl_xor(acc, m);
  __shared__ float red[4];
  if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = acc;
  __syncthreads();
  const float total = red[0] + red[1] + red[2] + red[3];
  const float inv = rsqrtf(total / (float)D + eps);
#pragma unroll
  for (int c = 0; c < 8; ++c) {
    const int i = threadIdx.x * 8 + c * 256 * 8;
    if (i < D) {
      ushort8 wv = *(const ushort8*)(w + i);
      ushort8 o;
#pragma unroll
      for (int j = 0; j < 8; ++j) o[j] = f2b(vals[c * 8 + j] * inv * (b2f(wv[j]) + w_bias));
      *(ushort8*)(out + off + i) = o;
    }
  }
}

// ---------------------------------------------------------------------------
// Fused RoPE (HF rotate-half) + KV-cache append, on the PACKED qkv tensor
// (one fused QKV GEMM writes [B, S, (H+2*KVH)*hd]; this kernel rotates the
// q heads in place, rotates k heads into the cache, copies v heads into the
// cache — no separate q/k/v tensors ever materialize).
// one wave per (b, s, head-slot); cache layout [B, KVH, T, hd];
// cos/sin tables fp32 [maxT, hd/2].
// ---------------------------------------------------------------------------

// When the MFMA-packed cache copies exist (kpc/vpc non-null, hd == 128) the
// same kernel also appends into them (decode attention then streams the
// cache as coalesced v_mfma_f32_16x16x32_bf16 B-fragments):
//   K_packed [B,KVH][T32/16 tile][4 hd-chunk][64 lane][8]  lane=(hd&31)/8*16 + (pos&15)
//   V_packed [B,KVH][8 hd-group][T32/32 tile][64 lane][8]  lane=((pos&31)>>3)*16 + (hd&15)
// Optional qwen3 per-head q/k RMSNorm (qn/kn weights [hd], fused before the
// rotation): the slot's wave reduces sum-of-squares over the head row with
// shfl_xor, then scales while rotating.
// fp8 packed mode (kp8 non-null): the packed copies are OCP e4m3 bytes with
// per-row scales sk/sv [B*KVH*T32] — half the decode stream and ~60% of the
// dual-cache residency (plain cache stays bf16 for prefill). XOT_FP8_KV=1.
__global__ __launch_bounds__(256) void rope_qkv_append_kernel(
    unsigned short* __restrict__ qkv, const float* __restrict__ cosb,
    const float* __restrict__ sinb, const int* __restrict__ positions,
    unsigned short* __restrict__ kc, unsigned short* __restrict__ vc,
    int B, int S, int H, int KVH, int hd, int T,
    unsigned short* __restrict__ kpc, unsigned short* __restrict__ vpc, int T32,
    const unsigned short* __restrict__ qn, const unsigned short* __restrict__ kn,
    float norm_eps, int npos,
    unsigned char* __restrict__ kp8, unsigned char* __restrict__ vp8,
    float* __restrict__ sk, float* __restrict__ sv) {
  const int wid = blockIdx.x * (blockDim.x >> 6) + (threadIdx.x >> 6);
  const int lane = threadIdx.x & 63;
  const int slots = H + 2 * KVH;
  if (wid >= B * S * slots) return;
  const int slot = wid % slots;
  const int bs = wid / slots;
  const int s = bs % S;
  const int b = bs / S;
  // positions: [S] (shared across batch) or [B*S] (per-row — continuous
  // batching where every slot decodes at its own position)
  const int pos = positions[(npos == B * S && npos != S) ? bs : s];
  const int hd2 = hd >> 1;
  unsigned short* row = qkv + ((size_t)bs * slots + slot) * hd;
  if (slot < H) {
    float x1 = 0.f, x2 = 0.f;
    if (lane < hd2) {
      x1 = b2f(row[lane]);
      x2 = b2f(row[lane + hd2]);
    }
    if (qn) {
      float ss = x1 * x1 + x2 * x2;
#pragma unroll
      for (int m = 32; m > 0; m >>= 1) ss += __shfl_xor(ss, m);
      const float inv = rsqrtf(ss / (float)hd + norm_eps);
      if (lane < hd2) {
        x1 *= inv * b2f(qn[lane]);
        x2 *= inv * b2f(qn[lane + hd2]);
      }
    }
    if (lane < hd2) {
      const float c = cosb[(size_t)pos * hd2 + lane];
      const float sn = sinb[(size_t)pos * hd2 + lane];
      row[lane] = f2b(x1 * c - x2 * sn);
      row[lane + hd2] = f2b(x2 * c + x1 * sn);
    }
  } else if (slot < H + KVH) {
    const int h = slot - H;
    unsigned short* dst = kc + (((size_t)(b * KVH + h) * T + pos) * hd);
    float kx1 = 0.f, kx2 = 0.f;
    if (lane < hd2) {
      kx1 = b2f(row[lane]);
      kx2 = b2f(row[lane + hd2]);
    }
    if (kn) {
      float ss = kx1 * kx1 + kx2 * kx2;
#pragma unroll
      for (int m = 32; m > 0; m >>= 1) ss += __shfl_xor(ss, m);
      const float inv = rsqrtf(ss / (float)hd + norm_eps);
      if (lane < hd2) {
        kx1 *= inv * b2f(kn[lane]);
        kx2 *= inv * b2f(kn[lane + hd2]);
      }
    }
    float f1 = 0.f, f2v = 0.f;
    {
      const float c = (lane < hd2) ? cosb[(size_t)pos * hd2 + lane] : 0.f;
      const float sn = (lane < hd2) ? sinb[(size_t)pos * hd2 + lane] : 0.f;
      f1 = kx1 * c - kx2 * sn;
      f2v = kx2 * c + kx1 * sn;
    }
    if (lane < hd2) {
      dst[lane] = f2b(f1);
      dst[lane + hd2] = f2b(f2v);
      if (kpc) {
        // packed K: element for hd-dim d at
        //   [(b*KVH+h)][pos>>4][d>>5][((d&31)>>3)*16 + (pos&15)][d&7]
        const size_t base = ((size_t)(b * KVH + h) * (T32 >> 4) + (pos >> 4)) * 2048;
        const int d1 = lane, d2 = lane + hd2;
        kpc[base + (size_t)(d1 >> 5) * 512 + (((d1 & 31) >> 3) * 16 + (pos & 15)) * 8 + (d1 & 7)] = f2b(f1);
        kpc[base + (size_t)(d2 >> 5) * 512 + (((d2 & 31) >> 3) * 16 + (pos & 15)) * 8 + (d2 & 7)] = f2b(f2v);
      }
    }
    if (kp8) {
      float mx = fmaxf(fabsf(f1), fabsf(f2v));
#pragma unroll
      for (int m = 32; m > 0; m >>= 1) mx = fmaxf(mx, __shfl_xor(mx, m));
      const float scl = fmaxf(mx, 1e-12f) / 448.f;
      const float inv = 1.f / scl;
      if (lane == 0) sk[(size_t)(b * KVH + h) * T32 + pos] = scl;
      if (lane < hd2) {
        const size_t base = ((size_t)(b * KVH + h) * (T32 >> 4) + (pos >> 4)) * 2048;
        const int d1 = lane, d2 = lane + hd2;
        const unsigned short p1 = (unsigned short)__builtin_amdgcn_cvt_pk_fp8_f32(f1 * inv, 0.f, 0, false);
        const unsigned short p2 = (unsigned short)__builtin_amdgcn_cvt_pk_fp8_f32(f2v * inv, 0.f, 0, false);
        kp8[base + (size_t)(d1 >> 5) * 512 + (((d1 & 31) >> 3) * 16 + (pos & 15)) * 8 + (d1 & 7)] = (unsigned char)(p1 & 0xff);
        kp8[base + (size_t)(d2 >> 5) * 512 + (((d2 & 31) >> 3) * 16 + (pos & 15)) * 8 + (d2 & 7)] = (unsigned char)(p2 & 0xff);
      }
    }
  } else {
    const int h = slot - H - KVH;
    unsigned short* dst = vc + (((size_t)(b * KVH + h) * T + pos) * hd);
    if (lane * 2 < hd)
      *(unsigned int*)(dst + lane * 2) = *(const unsigned int*)(row + lane * 2);
    if (vpc && lane * 2 < hd) {
      // packed V: element for hd-dim d at
      //   [(b*KVH+h)][d>>4][pos>>5][((pos&31)>>3)*16 + (d&15)][pos&7]
      const int tp = pos >> 5, qt = (pos & 31) >> 3, j = pos & 7;
      const size_t gbase = (size_t)(b * KVH + h) * 8;
#pragma unroll
      for (int e = 0; e < 2; ++e) {
        const int d = lane * 2 + e;
        vpc[((gbase + (d >> 4)) * (T32 >> 5) + tp) * 512 + (qt * 16 + (d & 15)) * 8 + j] = row[d];
      }
    }
    if (vp8) {
      float mx = 0.f;
      if (lane * 2 < hd) {
        mx = fmaxf(fabsf(b2f(row[lane * 2])), fabsf(b2f(row[lane * 2 + 1])));
      }
#pragma unroll
      for (int m = 32; m > 0; m >>= 1) mx = fmaxf(mx, __shfl_xor(mx, m));
      const float scl = fmaxf(mx, 1e-12f) / 448.f;
      const float inv = 1.f / scl;
      if (lane == 0) sv[(size_t)(b * KVH + h) * T32 + pos] = scl;
      if (lane * 2 < hd) {
        const int tp = pos >> 5, qt = (pos & 31) >> 3, j = pos & 7;
        const size_t gbase = (size_t)(b * KVH + h) * 8;
#pragma unroll
        for (int e = 0; e < 2; ++e) {
          const int d = lane * 2 + e;
          const unsigned short pk = (unsigned short)__builtin_amdgcn_cvt_pk_fp8_f32(b2f(row[d]) * inv, 0.f, 0, false);
          vp8[((gbase + (d >> 4)) * (T32 >> 5) + tp) * 512 + (qt * 16 + (d & 15)) * 8 + j] = (unsigned char)(pk & 0xff);
        }
      }
    }
  }
}

// ---------------------------------------------------------------------------
// GQA decode attention (flash-decoding): split-KV partials + merge.
//
// partial kernel: grid = B * KVH * NSPLIT workgroups, 256 threads = 4 waves
// = 16 groups of 16 lanes. Each group walks cache positions with stride 16;
// a group handles one position per step: 16 lanes x 16 B = one 256 B KV row
// (hd=128) coalesced. All NQ = H/KVH query heads of this kv-head are scored
// in the same pass (KV bytes read once per kv-head). Online softmax per
// (group, head); group partials merged through LDS; one (m, l, o[hd]) fp32
// partial per (b, qh, split) written to the workspace.
// ---------------------------------------------------------------------------

template <int NQ, int HD>
__global__ __launch_bounds__(256) void attn_decode_partial(
    const unsigned short* __restrict__ q, const unsigned short* __restrict__ kc,
    const unsigned short* __restrict__ vc, const int* __restrict__ seq_lens,
    float* __restrict__ ws_o, float* __restrict__ ws_ml,
    int B, int H, int KVH, int T, int nsplit, int qh0, float scale, long long q_stride) {
  constexpr int EPL = HD / 16;  // bf16 elements per lane (8 @128, 4 @64)
  const int blk = blockIdx.x;
  const int split = blk % nsplit;
  const int t1 = blk / nsplit;
  const int kvh = t1 % KVH;
  const int b = t1 / KVH;
  const int sl = seq_lens[b];
  const int chunk = (T + nsplit - 1) / nsplit;  // capacity-static (graph-safe)
  const int c0 = split * chunk;
  const int c1 = min(c0 + chunk, sl);
  const int lane = threadIdx.x & 63;
  const int gl = lane & 15;
  const int group = (threadIdx.x >> 6) * 4 + (lane >> 4);  // 0..15

  const int qh_base = kvh * (H / KVH) + qh0;
  float qreg[NQ][EPL];
#pragma unroll
  for (int n = 0; n < NQ; ++n) {
    const unsigned short* qp = q + ((size_t)b * q_stride + (qh_base + n) * HD + gl * EPL);
#pragma unroll
    for (int e = 0; e < EPL; ++e) qreg[n][e] = b2f(qp[e]) * scale;
  }

  float m[NQ], l[NQ], oacc[NQ][EPL];
#pragma unroll
  for (int n = 0; n < NQ; ++n) {
    m[n] = -INFINITY;
    l[n] = 0.f;
#pragma unroll
    for (int e = 0; e < EPL; ++e) oacc[n][e] = 0.f;
  }

  const size_t cache_base = ((size_t)(b * KVH + kvh)) * T * HD;
  for (int t = c0 + group; t < c1; t += 16) {
    float kf[EPL], vf[EPL];
    {
      const unsigned short* kr = kc + cache_base + (size_t)t * HD + gl * EPL;
      const unsigned short* vr = vc + cache_base + (size_t)t * HD + gl * EPL;
      if constexpr (EPL == 8) {
        ushort8 kv8 = *(const ushort8*)kr;
        ushort8 vv8 = *(const ushort8*)vr;
#pragma unroll
        for (int e = 0; e < 8; ++e) { kf[e] = b2f(kv8[e]); vf[e] = b2f(vv8[e]); }
      } else {
        ushort4_t kv4 = *(const ushort4_t*)kr;
        ushort4_t vv4 = *(const ushort4_t*)vr;
#pragma unroll
        for (int e = 0; e < 4; ++e) { kf[e] = b2f(kv4[e]); vf[e] = b2f(vv4[e]); }
      }
    }
    float dot[NQ];
#pragma unroll
    for (int n = 0; n < NQ; ++n) {
      float d = 0.f;
#pragma unroll
      for (int e = 0; e < EPL; ++e) d += qreg[n][e] * kf[e];
      dot[n] = d;
    }
    // reduce the dot across the 16-lane group (xor masks < 16 stay in-group)
#pragma unroll
    for (int n = 0; n < NQ; ++n) {
#pragma unroll
      for (int mm = 8; mm > 0; mm >>= 1) dot[n] += __shfl_xor(dot[n], mm);
    }
#pragma unroll
    for (int n = 0; n < NQ; ++n) {
      const float s = dot[n];
      const float mn = fmaxf(m[n], s);
      const float alpha = (l[n] > 0.f) ? __expf(m[n] - mn) : 0.f;
      const float p = __expf(s - mn);
      l[n] = l[n] * alpha + p;
#pragma unroll
      for (int e = 0; e < EPL; ++e) oacc[n][e] = oacc[n][e] * alpha + p * vf[e];
      m[n] = mn;
    }
  }

  // merge the 16 group-partials through LDS -> one partial per (head, split)
  __shared__ float lds_o[16 * NQ * HD];
  __shared__ float lds_ml[16 * NQ * 2];
#pragma unroll
  for (int n = 0; n < NQ; ++n) {
#pragma unroll
    for (int e = 0; e < EPL; ++e) lds_o[(group * NQ + n) * HD + gl * EPL + e] = oacc[n][e];
    if (gl == 0) {
      lds_ml[(group * NQ + n) * 2 + 0] = m[n];
      lds_ml[(group * NQ + n) * 2 + 1] = l[n];
    }
  }
  __syncthreads();
  // 256 threads; HD (<=128) of them combine the 16 groups per head
  for (int n = 0; n < NQ; ++n) {
    const int d = threadIdx.x;
    if (d < HD) {
      float M = -INFINITY;
#pragma unroll
      for (int g = 0; g < 16; ++g) M = fmaxf(M, lds_ml[(g * NQ + n) * 2 + 0]);
      float L = 0.f, O = 0.f;
#pragma unroll
      for (int g = 0; g < 16; ++g) {
        const float lg = lds_ml[(g * NQ + n) * 2 + 1];
        const float alpha = (lg > 0.f) ? __expf(lds_ml[(g * NQ + n) * 2 + 0] - M) : 0.f;
        L += alpha * lg;
        O += alpha * lds_o[(g * NQ + n) * HD + d];
      }
      const int qh = qh_base + n;
      const size_t pidx = ((size_t)(b * H + qh) * nsplit + split);
      ws_o[pidx * HD + d] = O;
      if (d == 0) {
        ws_ml[pidx * 2 + 0] = M;
        ws_ml[pidx * 2 + 1] = L;
      }
    }
  }
}

// ---------------------------------------------------------------------------
// MFMA flash-decoding attention (hd = 128): scores and PV on matrix cores.
//
// One WAVE per (b, kv-head, kv-split); the wave's all NQ (<=16) query heads
// are scored together: per 32-position tile,
//   scores[16q][32p] = 2 x (4 x v_mfma_f32_16x16x32_bf16)  (Q fragments resident,
//                      K streamed from the packed cache as coalesced 1 KB loads)
//   online softmax row stats via 4 shfl_xor over the 16-lane column groups
//   P -> bf16 A-fragments through a 96 B-stride LDS image (conflict-free)
//   out[16q][128] += 8 x v_mfma_f32_16x16x32_bf16 (V streamed packed)
// No cross-wave barriers (per-wave LDS slice), so ragged per-batch lengths
// cannot deadlock. Partials go to the same (m, l, o) workspace as the VALU
// kernel and are merged by attn_decode_merge<128>.
// Replaces the torchtune cached-decode step (reference general_mha.py:211-215);
// the VALU split-KV kernel above stays as the hd=64 / unpacked-cache path.
// ---------------------------------------------------------------------------

// softcap > 0 applies gemma2's attention-logit soft-capping
// (s = cap * tanh(s / cap), after scale, before masking); window > 0 is the
// sliding-window mask (query at sl-1 sees positions [sl - window, sl)).
// Both are wave-uniform runtime flags: the llama path (0, 0) takes no tanh.
// FP8: the packed cache copies are OCP e4m3 bytes with per-row scales
// sk/sv (appended by rope_qkv_append's fp8 mode) — half the stream bytes.
// q is quantized per head in-kernel; scores rescale by s_q[row]*s_k[col];
// PV keeps a per-tile running scale R (s_v folded into the quantized P).
template <bool PREFETCH = false, bool FP8 = false>
__global__ __launch_bounds__(256) void attn_decode_mfma_kernel(
    const unsigned short* __restrict__ q, const unsigned short* __restrict__ kp,
    const unsigned short* __restrict__ vp, const int* __restrict__ seq_lens,
    float* __restrict__ ws_o, float* __restrict__ ws_ml,
    int B, int H, int KVH, int T32, int nsplit, float scale, long long q_stride,
    float softcap, int window,
    const float* __restrict__ sk = nullptr, const float* __restrict__ sv = nullptr) {
  const int wv = threadIdx.x >> 6;
  const int wid = blockIdx.x * 4 + wv;
  __shared__ unsigned short plds_all[4][16 * 48];  // 96 B row stride: bank-conflict-free b128 reads
  if (wid >= B * KVH * nsplit) return;
  const int split = wid % nsplit;
  const int kvh = (wid / nsplit) % KVH;
  const int b = wid / (nsplit * KVH);
  const int lane = threadIdx.x & 63;
  const int NQ = H / KVH;
  const int sl = seq_lens[b];
  const int chunk = ((T32 / nsplit + 31) >> 5) << 5;
  const int win_lo = (window > 0) ? max(0, sl - window) : 0;  // first visible pos
  const int c0 = max(split * chunk, (win_lo >> 5) << 5);
  const int c1 = min(split * chunk + chunk, sl);
  unsigned short* plds = plds_all[wv];

  // Q fragments: A[i = lane&15 (query head, clamped), k = (lane>>4)*8 + j]
  const int qh_base = kvh * NQ;
  const int qi = min(lane & 15, NQ - 1);
  bf16x8 qf[4];
  {
    const unsigned short* qrow = q + (size_t)b * q_stride + (size_t)(qh_base + qi) * 128;
#pragma unroll
    for (int c = 0; c < 4; ++c)
      qf[c] = *reinterpret_cast<const bf16x8*>(qrow + c * 32 + (lane >> 4) * 8);
  }
  long qf8[4];
  float srow[4];
  if (FP8) {
    float mx = 0.f;
#pragma unroll
    for (int c = 0; c < 4; ++c)
#pragma unroll
      for (int j = 0; j < 8; ++j) mx = fmaxf(mx, fabsf((float)qf[c][j]));
    mx = fmaxf(mx, __shfl_xor(mx, 16));
    mx = fmaxf(mx, __shfl_xor(mx, 32));
    const float sq = fmaxf(mx, 1e-12f) / 448.f;
    const float inv = 1.f / sq;
#pragma unroll
    for (int c = 0; c < 4; ++c) {
      unsigned char o[8];
#pragma unroll
      for (int j = 0; j < 8; j += 2) {
        const unsigned short pk = (unsigned short)__builtin_amdgcn_cvt_pk_fp8_f32(
            (float)qf[c][j] * inv, (float)qf[c][j + 1] * inv, 0, false);
        o[j] = (unsigned char)(pk & 0xff);
        o[j + 1] = (unsigned char)(pk >> 8);
      }
      qf8[c] = *reinterpret_cast<const long*>(o);
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) srow[r] = __shfl(sq, (lane >> 4) * 4 + r);
  }

  float m[4], lsum[4];
  floatx4 acco[8];
#pragma unroll
  for (int r = 0; r < 4; ++r) { m[r] = -INFINITY; lsum[r] = 0.f; }
#pragma unroll
  for (int g = 0; g < 8; ++g) acco[g] = (floatx4)(0.f);

  const size_t kbase = (size_t)(b * KVH + kvh) * (T32 >> 4) * 2048;
  const size_t vbase = (size_t)(b * KVH + kvh) * 8 * (T32 >> 5) * 512;
  const int col = lane & 15;

  // PREFETCH: the next tile's 8 K fragments are loaded during the previous
  // tile's PV phase (kbuf registers, +32 VGPR) so the score MFMAs never
  // wait on HBM; measured A/B via XOT_ATTN_PREFETCH.
  bf16x8 kbuf[8];
  long kbuf8[8];
  const unsigned char* kp8 = reinterpret_cast<const unsigned char*>(kp);
  const unsigned char* vp8 = reinterpret_cast<const unsigned char*>(vp);
  const size_t ssbase = (size_t)(b * KVH + kvh) * T32;
  float Rscale = 1.f;
  if (PREFETCH && c0 < c1) {
#pragma unroll
    for (int h = 0; h < 2; ++h) {
      if (FP8) {
        const unsigned char* kt = kp8 + kbase + ((size_t)((c0 >> 4) + h)) * 2048 + (size_t)lane * 8;
#pragma unroll
        for (int c = 0; c < 4; ++c)
          kbuf8[h * 4 + c] = __builtin_nontemporal_load(reinterpret_cast<const long*>(kt + c * 512));
      } else {
        const unsigned short* kt = kp + kbase + ((size_t)((c0 >> 4) + h)) * 2048 + (size_t)lane * 8;
#pragma unroll
        for (int c = 0; c < 4; ++c)
          kbuf[h * 4 + c] = __builtin_nontemporal_load(reinterpret_cast<const bf16x8*>(kt + c * 512));
      }
    }
  }

  for (int t = c0; t < c1; t += 32) {
    // ---- scores: two 16-position half-tiles ----
    floatx4 sc[2];
#pragma unroll
    for (int h = 0; h < 2; ++h) {
      sc[h] = (floatx4)(0.f);
      if (FP8) {
        const unsigned char* kt = kp8 + kbase + ((size_t)((t >> 4) + h)) * 2048 + (size_t)lane * 8;
#pragma unroll
        for (int c = 0; c < 4; ++c) {
          const long kb = PREFETCH ? kbuf8[h * 4 + c]
              : __builtin_nontemporal_load(reinterpret_cast<const long*>(kt + c * 512));
          sc[h] = __builtin_amdgcn_mfma_f32_16x16x32_fp8_fp8(qf8[c], kb, sc[h], 0, 0, 0);
        }
      } else {
        const unsigned short* kt = kp + kbase + ((size_t)((t >> 4) + h)) * 2048 + (size_t)lane * 8;
#pragma unroll
        for (int c = 0; c < 4; ++c) {
          const bf16x8 kb = PREFETCH ? kbuf[h * 4 + c]
              : __builtin_nontemporal_load(reinterpret_cast<const bf16x8*>(kt + c * 512));
          sc[h] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(qf[c], kb, sc[h], 0, 0, 0);
        }
      }
    }
    // ---- online softmax (rows r are this lane's 4 query heads) ----
    float rmax[4];
#pragma unroll
    for (int h = 0; h < 2; ++h) {
      const int pos = t + h * 16 + col;
      const bool ok = pos < c1 && pos >= win_lo;
      const float skc = FP8 ? sk[ssbase + min(pos, T32 - 1)] : 1.f;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        float s = sc[h][r] * scale;
        if (FP8) s *= srow[r] * skc;
        if (softcap > 0.f) s = softcap * tanhf(s * (1.f / softcap));
        sc[h][r] = ok ? s : -INFINITY;
      }
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) rmax[r] = fmaxf(sc[0][r], sc[1][r]);
#pragma unroll
    for (int mm = 1; mm < 16; mm <<= 1)
#pragma unroll
      for (int r = 0; r < 4; ++r) rmax[r] = fmaxf(rmax[r], __shfl_xor(rmax[r], mm));
    float alpha[4], rsum[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const float mn = fmaxf(m[r], rmax[r]);
      alpha[r] = (lsum[r] > 0.f) ? __expf(m[r] - mn) : 0.f;
      m[r] = mn;
      float p0 = __expf(sc[0][r] - mn);
      float p1 = __expf(sc[1][r] - mn);
      sc[0][r] = p0;
      sc[1][r] = p1;
      rsum[r] = p0 + p1;
    }
#pragma unroll
    for (int mm = 1; mm < 16; mm <<= 1)
#pragma unroll
      for (int r = 0; r < 4; ++r) rsum[r] += __shfl_xor(rsum[r], mm);
#pragma unroll
    for (int r = 0; r < 4; ++r) lsum[r] = lsum[r] * alpha[r] + rsum[r];
    float s_pv = 1.f, rfac = 1.f;
    if (FP8) {
      // per-tile V scale ceiling; acco is kept in units of 1/R so quantized
      // P' = p * s_v[pos] / s_pv enters at full e4m3 range
      float mv = sv[ssbase + min(t + (lane & 31), T32 - 1)];
#pragma unroll
      for (int m_ = 32; m_ > 0; m_ >>= 1) mv = fmaxf(mv, __shfl_xor(mv, m_));
      s_pv = fmaxf(mv, 1e-12f);
      rfac = Rscale / s_pv;
      Rscale = s_pv;
    }
#pragma unroll
    for (int g = 0; g < 8; ++g)
#pragma unroll
      for (int r = 0; r < 4; ++r) acco[g][r] *= alpha[r] * (FP8 ? rfac : 1.f);
    // ---- P -> LDS (bf16 / fp8 bytes, conflict-padded) and back as A fragments ----
    long pf8 = 0;
    bf16x8 pf;
    if (FP8) {
      unsigned char* pl8 = reinterpret_cast<unsigned char*>(plds);
#pragma unroll
      for (int h = 0; h < 2; ++h) {
        const int pos = t + h * 16 + col;
        const float svv = sv[ssbase + min(pos, T32 - 1)];
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const unsigned short pk = (unsigned short)__builtin_amdgcn_cvt_pk_fp8_f32(
              sc[h][r] * svv / s_pv, 0.f, 0, false);
          pl8[((lane >> 4) * 4 + r) * 48 + h * 16 + col] = (unsigned char)(pk & 0xff);
        }
      }
      pf8 = *reinterpret_cast<const long*>(pl8 + (lane & 15) * 48 + (lane >> 4) * 8);
    } else {
#pragma unroll
      for (int h = 0; h < 2; ++h)
#pragma unroll
        for (int r = 0; r < 4; ++r)
          plds[((lane >> 4) * 4 + r) * 48 + h * 16 + col] = f2b(sc[h][r]);
      pf = *reinterpret_cast<const bf16x8*>(plds + (lane & 15) * 48 + (lane >> 4) * 8);
    }
    if (PREFETCH && t + 32 < c1) {
      // issue next tile's K stream now; it completes under the PV MFMAs
#pragma unroll
      for (int h = 0; h < 2; ++h) {
        if (FP8) {
          const unsigned char* kt = kp8 + kbase + ((size_t)(((t + 32) >> 4) + h)) * 2048 + (size_t)lane * 8;
#pragma unroll
          for (int c = 0; c < 4; ++c)
            kbuf8[h * 4 + c] = __builtin_nontemporal_load(reinterpret_cast<const long*>(kt + c * 512));
        } else {
          const unsigned short* kt = kp + kbase + ((size_t)(((t + 32) >> 4) + h)) * 2048 + (size_t)lane * 8;
#pragma unroll
          for (int c = 0; c < 4; ++c)
            kbuf[h * 4 + c] = __builtin_nontemporal_load(reinterpret_cast<const bf16x8*>(kt + c * 512));
        }
      }
    }
    // ---- PV: out[16q][g*16..] += P x V ----
    if (FP8) {
      const unsigned char* vt = vp8 + vbase + (size_t)(t >> 5) * 512 + (size_t)lane * 8;
#pragma unroll
      for (int g = 0; g < 8; ++g) {
        const long vb = __builtin_nontemporal_load(
            reinterpret_cast<const long*>(vt + (size_t)g * (T32 >> 5) * 512));
        acco[g] = __builtin_amdgcn_mfma_f32_16x16x32_fp8_fp8(pf8, vb, acco[g], 0, 0, 0);
      }
    } else {
      const unsigned short* vt = vp + vbase + (size_t)(t >> 5) * 512 + (size_t)lane * 8;
#pragma unroll
      for (int g = 0; g < 8; ++g) {
        const bf16x8 vb = __builtin_nontemporal_load(
            reinterpret_cast<const bf16x8*>(vt + (size_t)g * (T32 >> 5) * 512));
        acco[g] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(pf, vb, acco[g], 0, 0, 0);
      }
    }
  }

  // ---- epilogue: one (m, l, o[128]) partial per (b, qh, split) ----
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int qrow = (lane >> 4) * 4 + r;
    if (qrow < NQ) {
      const size_t pidx = ((size_t)(b * H + qh_base + qrow) * nsplit + split);
#pragma unroll
      for (int g = 0; g < 8; ++g) ws_o[pidx * 128 + g * 16 + col] = acco[g][r] * (FP8 ? Rscale : 1.f);
      if (col == 0) {
        ws_ml[pidx * 2 + 0] = m[r];
        ws_ml[pidx * 2 + 1] = lsum[r];
      }
    }
  }
}

// ---------------------------------------------------------------------------
// MFMA flash-forward prefill attention (hd = 128, causal, GQA).
//
// Replaces torch sdpa for the prefill step (reference: torchtune
// MultiHeadAttention prefill, general_mha.py:218-226; sdpa measures ~1.8 ms
// per 70B layer at B=64xS=512 — VALU/flash at ~300 TF).  Grid: one 4-wave
// workgroup per (b, q-head, 128-row q block); the block's waves share K/V
// tiles staged in LDS from the MFMA-packed cache (fragment layout is
// lane-linear, so staging is 1 KB coalesced loads and conflict-free b128
// reads).  Each wave owns 32 q rows (2 MFMA sub-tiles), walks kv position
// tiles of 32 with online softmax, masks the causal boundary, writes final
// bf16 rows (no split-K workspace).
// ---------------------------------------------------------------------------

__global__ __launch_bounds__(256) void attn_prefill_mfma_kernel(
    const unsigned short* __restrict__ q, const unsigned short* __restrict__ kp,
    const unsigned short* __restrict__ vp, unsigned short* __restrict__ out,
    int B, int S, int H, int KVH, int T32, int start_pos,
    long long q_bstride, long long q_sstride, float scale,
    float softcap, int window) {
  // block -> (b, h, q-block)
  const int qblocks = (S + 127) >> 7;
  const int h = blockIdx.x % H;
  const int t1 = blockIdx.x / H;
  const int qb = t1 % qblocks;
  const int b = t1 / qblocks;
  const int wv = threadIdx.x >> 6;
  const int lane = threadIdx.x & 63;
  const int kvh = h / (H / KVH);

  // this wave's 32 q rows: [r0, r0+32)
  const int r0 = qb * 128 + wv * 32;
  const int col = lane & 15;

  __shared__ unsigned short kv_lds[2][8192];  // K tile 8 KB + V tile 8 KB, dbuf

  // Q fragments for 2 sub-tiles x 4 hd-chunks; rows clamped to S-1 (writes
  // are predicated, extra rows only waste compute)
  bf16x8 qf[2][4];
#pragma unroll
  for (int t = 0; t < 2; ++t) {
    const int row = min(r0 + t * 16 + col, S - 1);
    const unsigned short* qrow = q + (size_t)b * q_bstride + (size_t)row * q_sstride + (size_t)h * 128;
#pragma unroll
    for (int c = 0; c < 4; ++c)
      qf[t][c] = *reinterpret_cast<const bf16x8*>(qrow + c * 32 + (lane >> 4) * 8);
  }

  float m[2][4], lsum[2][4];
  floatx4 acco[2][8];
#pragma unroll
  for (int t = 0; t < 2; ++t)
#pragma unroll
    for (int r = 0; r < 4; ++r) { m[t][r] = -INFINITY; lsum[t][r] = 0.f; }
#pragma unroll
  for (int t = 0; t < 2; ++t)
#pragma unroll
    for (int g = 0; g < 8; ++g) acco[t][g] = (floatx4)(0.f);

  const size_t kbase = (size_t)(b * KVH + kvh) * (T32 >> 4) * 2048;
  const size_t vbase = (size_t)(b * KVH + kvh) * 8 * (T32 >> 5) * 512;
  // causal end for the BLOCK (max row): positions [0, start_pos + block_hi]
  const int block_hi = min(qb * 128 + 127, S - 1);
  const int kv_end = start_pos + block_hi + 1;  // exclusive

  __shared__ unsigned short plds_all[4][16 * 48 * 2];

  // cooperative stage of kv tile `tp` (32 positions) into kv_lds[buf]
  auto stage = [&](int tp, int buf) {
    // K: two 16-pos tiles x 4 chunks x 512 elems; V: 8 groups x 512 elems
    // 256 threads x 24 pieces of 256 B... simpler: each thread copies 16 B x3
    const unsigned short* ksrc = kp + kbase + (size_t)(tp * 2) * 2048;
    const unsigned short* vsrc = vp + vbase + (size_t)tp * 512;
    unsigned short* dk = kv_lds[buf];
    unsigned short* dv = kv_lds[buf] + 4096;
    const int tid = threadIdx.x;
    // K: 4096 elems = 8192 B: 256 threads x 2 x 16 B
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      const int e = (tid + i * 256) * 8;
      *(ushort8*)(dk + e) = *(const ushort8*)(ksrc + e);
    }
    // V: 8 groups x 512 elems, group stride (T32>>5)*512 in global
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      const int e = tid + i * 256;           // 0..511 -> (group, piece)
      const int g = e >> 6, piece = e & 63;  // 64 pieces of 8 elems per group
      *(ushort8*)(dv + g * 512 + piece * 8) =
          *(const ushort8*)(vsrc + (size_t)g * (T32 >> 5) * 512 + piece * 8);
    }
  };

  const int ntiles = (kv_end + 31) >> 5;
  // sliding window: the block's lowest q row sees nothing before
  // start_pos + qb*128 - window + 1 — skip whole kv tiles below it
  const int tp0 = (window > 0) ? max(0, (start_pos + qb * 128 - window + 1) >> 5) : 0;
  stage(tp0, tp0 & 1);
  __syncthreads();

  for (int tp = tp0; tp < ntiles; ++tp) {
    const int buf = tp & 1;
    if (tp + 1 < ntiles) stage(tp + 1, buf ^ 1);  // plain loads overlap compute
    const unsigned short* dk = kv_lds[buf];
    const unsigned short* dv = kv_lds[buf] + 4096;
    unsigned short* plds = plds_all[wv];
#pragma unroll
    for (int t = 0; t < 2; ++t) {
      // scores for two 16-pos halves of this kv tile
      floatx4 sc[2];
#pragma unroll
      for (int hh = 0; hh < 2; ++hh) {
        sc[hh] = (floatx4)(0.f);
#pragma unroll
        for (int c = 0; c < 4; ++c) {
          const bf16x8 kb = *reinterpret_cast<const bf16x8*>(dk + (hh * 4 + c) * 512 + lane * 8);
          sc[hh] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(qf[t][c], kb, sc[hh], 0, 0, 0);
        }
      }
      // causal mask: kv pos must be < start_pos + row + 1
      float rmax[4];
#pragma unroll
      for (int hh = 0; hh < 2; ++hh) {
        const int pos = tp * 32 + hh * 16 + col;
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int row = r0 + t * 16 + (lane >> 4) * 4 + r;
          bool ok = (pos <= start_pos + row) && (pos < kv_end);
          if (window > 0) ok = ok && (pos > start_pos + row - window);
          float s = sc[hh][r] * scale;
          if (softcap > 0.f) s = softcap * tanhf(s * (1.f / softcap));
          sc[hh][r] = ok ? s : -INFINITY;
        }
      }
#pragma unroll
      for (int r = 0; r < 4; ++r) rmax[r] = fmaxf(sc[0][r], sc[1][r]);
#pragma unroll
      for (int mm = 1; mm < 16; mm <<= 1)
#pragma unroll
        for (int r = 0; r < 4; ++r) rmax[r] = fmaxf(rmax[r], __shfl_xor(rmax[r], mm));
      float alpha[4], rsum[4];
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const float mn = fmaxf(m[t][r], rmax[r]);
        if (mn == -INFINITY) { alpha[r] = 1.f; rsum[r] = 0.f; sc[0][r] = 0.f; sc[1][r] = 0.f; continue; }
        alpha[r] = (lsum[t][r] > 0.f) ? __expf(m[t][r] - mn) : 0.f;
        m[t][r] = mn;
        const float p0 = __expf(sc[0][r] - mn);
        const float p1 = __expf(sc[1][r] - mn);
        sc[0][r] = p0;
        sc[1][r] = p1;
        rsum[r] = p0 + p1;
      }
#pragma unroll
      for (int mm = 1; mm < 16; mm <<= 1)
#pragma unroll
        for (int r = 0; r < 4; ++r) rsum[r] += __shfl_xor(rsum[r], mm);
#pragma unroll
      for (int r = 0; r < 4; ++r) lsum[t][r] = lsum[t][r] * alpha[r] + rsum[r];
#pragma unroll
      for (int g = 0; g < 8; ++g)
#pragma unroll
        for (int r = 0; r < 4; ++r) acco[t][g][r] *= alpha[r];
      unsigned short* pl = plds + t * 16 * 48;  // reuse the 2x buffer per sub-tile
#pragma unroll
      for (int hh = 0; hh < 2; ++hh)
#pragma unroll
        for (int r = 0; r < 4; ++r)
          pl[((lane >> 4) * 4 + r) * 48 + hh * 16 + col] = f2b(sc[hh][r]);
      const bf16x8 pf = *reinterpret_cast<const bf16x8*>(pl + (lane & 15) * 48 + (lane >> 4) * 8);
#pragma unroll
      for (int g = 0; g < 8; ++g) {
        const bf16x8 vb = *reinterpret_cast<const bf16x8*>(dv + g * 512 + lane * 8);
        acco[t][g] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(pf, vb, acco[t][g], 0, 0, 0);
      }
    }
    __syncthreads();  // all waves done with kv_lds[buf] before restaging
  }

  // epilogue: out[b, row, h, g*16 + col] = acc / lsum
#pragma unroll
  for (int t = 0; t < 2; ++t) {
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int row = r0 + t * 16 + (lane >> 4) * 4 + r;
      if (row < S) {
        const float inv = (lsum[t][r] > 0.f) ? 1.f / lsum[t][r] : 0.f;
        unsigned short* orow = out + (((size_t)b * S + row) * H + h) * 128;
#pragma unroll
        for (int g = 0; g < 8; ++g) orow[g * 16 + col] = f2b(acco[t][g][r] * inv);
      }
    }
  }
}

// layout probe for tests: one v_mfma_f32_16x16x32_bf16, row-major inputs
__global__ void mfma16_probe_kernel(const unsigned short* __restrict__ A,
                                    const unsigned short* __restrict__ Bm,
                                    float* __restrict__ D) {
  const int lane = threadIdx.x;
  bf16x8 a = *reinterpret_cast<const bf16x8*>(A + (lane & 15) * 32 + (lane >> 4) * 8);
  bf16x8 b;
#pragma unroll
  for (int j = 0; j < 8; ++j) b[j] = *reinterpret_cast<const __bf16*>(Bm + ((lane >> 4) * 8 + j) * 16 + (lane & 15));
  floatx4 d = (floatx4)(0.f);
  d = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, d, 0, 0, 0);
#pragma unroll
  for (int r = 0; r < 4; ++r) D[((lane >> 4) * 4 + r) * 16 + (lane & 15)] = d[r];
}

template <int HD>
__global__ __launch_bounds__(128) void attn_decode_merge(
    const float* __restrict__ ws_o, const float* __restrict__ ws_ml,
    unsigned short* __restrict__ out, int nsplit) {
  const int bh = blockIdx.x;  // b * H + qh
  const int d = threadIdx.x;
  if (d >= HD) return;
  float M = -INFINITY;
  for (int i = 0; i < nsplit; ++i) M = fmaxf(M, ws_ml[((size_t)bh * nsplit + i) * 2 + 0]);
  float L = 0.f, O = 0.f;
  for (int i = 0; i < nsplit; ++i) {
    const float lg = ws_ml[((size_t)bh * nsplit + i) * 2 + 1];
    const float alpha = (lg > 0.f) ? __expf(ws_ml[((size_t)bh * nsplit + i) * 2 + 0] - M) : 0.f;
    L += alpha * lg;
    O += alpha * ws_o[((size_t)bh * nsplit + i) * HD + d];
  }
  out[(size_t)bh * HD + d] = f2b(L > 0.f ? O / L : 0.f);
}

// ---------------------------------------------------------------------------
// MoE decode-routing glue: the static-capacity routed path needs
// (token-expert pairs -> per-expert-sorted gather list) and the weighted
// combine. In torch this is ~8 launches per MoE layer per step (argsort,
// repeat_interleave, cumsum, eq+sum, clamp, where, index_add) — measured as
// the TOP decode cost on DeepSeek-V2-Lite (profiles/r02_new_decoders_...).
// Here: ONE single-workgroup counting-sort kernel (A = T*k pairs <= 2048,
// E <= 256 fits LDS) + ONE deterministic gather-combine kernel (no atomics:
// out[t] = sum_j w[t,j] * y[pos(t,j)]).
// ---------------------------------------------------------------------------

// Fused MoE router: one wave per token row over the gate logits [T, E].
// mode 0: softmax -> top-k -> renormalize (Mixtral / qwen3-moe).
// mode 1: sigmoid + e-score bias -> group-limited top-k (top-2-sum group
//         scores, keep topk_group groups) -> gather sigmoid weights ->
//         optional renorm -> routed scaling (DeepSeek V2/V3).
// Replaces ~4-10 torch launches per MoE layer per step. E <= 256, k <= 8.
__global__ __launch_bounds__(256) void moe_route_kernel(
    const float* __restrict__ logits, const float* __restrict__ bias,
    int* __restrict__ idx, float* __restrict__ w,
    int T, int E, int k, int mode, int n_group, int topk_group,
    float routed_scale, int norm_topk) {
  const int row = blockIdx.x * (blockDim.x >> 6) + (threadIdx.x >> 6);
  if (row >= T) return;
  const int lane = threadIdx.x & 63;
  // per-lane 4 contiguous elements (E <= 256)
  float v[4], s[4], c[4];
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    const int e = lane * 4 + j;
    v[j] = (e < E) ? logits[(size_t)row * E + e] : -INFINITY;
  }
  if (mode == 0) {
    // softmax over the row
    float mx = fmaxf(fmaxf(v[0], v[1]), fmaxf(v[2], v[3]));
#pragma unroll
    for (int m = 32; m > 0; m >>= 1) mx = fmaxf(mx, __shfl_xor(mx, m));
    float sum = 0.f;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      s[j] = (v[j] == -INFINITY) ? 0.f : __expf(v[j] - mx);
      sum += s[j];
    }
#pragma unroll
    for (int m = 32; m > 0; m >>= 1) sum += __shfl_xor(sum, m);
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      s[j] /= sum;
      c[j] = (v[j] == -INFINITY) ? -INFINITY : s[j];
    }
  } else {
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      s[j] = 1.f / (1.f + __expf(-v[j]));
      const int e = lane * 4 + j;
      c[j] = (e < E) ? s[j] + (bias ? bias[e] : 0.f) : -INFINITY;
    }
    if (n_group > 1) {
      // group score = sum of top-2 choice values in the group; keep the
      // topk_group best groups, mask the rest
      const int gsize = E / n_group;  // elements per group (>= 4 assumed)
      float gs[8];
      for (int g = 0; g < n_group; ++g) {
        float m1 = -INFINITY, m2 = -INFINITY;
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          const int e = lane * 4 + j;
          const float cv = (e >= g * gsize && e < (g + 1) * gsize) ? c[j] : -INFINITY;
          if (cv > m1) { m2 = m1; m1 = cv; }
          else if (cv > m2) { m2 = cv; }
        }
        // wave-combine per-lane top2
#pragma unroll
        for (int m = 32; m > 0; m >>= 1) {
          const float o1 = __shfl_xor(m1, m);
          const float o2 = __shfl_xor(m2, m);
          if (o1 > m1) { m2 = fmaxf(m1, o2); m1 = o1; }
          else { m2 = fmaxf(m2, o1); }
        }
        gs[g] = m1 + (m2 == -INFINITY ? 0.f : m2);
      }
      // select topk_group groups (all lanes hold identical gs)
      unsigned int keep = 0;
      for (int t = 0; t < topk_group; ++t) {
        int best = -1;
        float bv = -INFINITY;
        for (int g = 0; g < n_group; ++g)
          if (!(keep >> g & 1) && gs[g] > bv) { bv = gs[g]; best = g; }
        if (best >= 0) keep |= 1u << best;
      }
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const int e = lane * 4 + j;
        if (e < E && !(keep >> (e / gsize) & 1)) c[j] = -INFINITY;
      }
    }
  }
  // iterative wave-wide top-k on c; weights come from s
  float wsum = 0.f;
  float wk[8];
  int ik[8];
  for (int t = 0; t < k; ++t) {
    float mx = fmaxf(fmaxf(c[0], c[1]), fmaxf(c[2], c[3]));
#pragma unroll
    for (int m = 32; m > 0; m >>= 1) mx = fmaxf(mx, __shfl_xor(mx, m));
    // lowest index attaining the max (torch.topk tie convention)
    int my = INT_MAX;
#pragma unroll
    for (int j = 0; j < 4; ++j)
      if (c[j] == mx && lane * 4 + j < my) my = lane * 4 + j;
#pragma unroll
    for (int m = 32; m > 0; m >>= 1) my = min(my, __shfl_xor(my, m));
    const int owner = my >> 2, slot = my & 3;
    float sv;
    switch (slot) {
      case 0: sv = __shfl(s[0], owner); break;
      case 1: sv = __shfl(s[1], owner); break;
      case 2: sv = __shfl(s[2], owner); break;
      default: sv = __shfl(s[3], owner); break;
    }
    ik[t] = my;
    wk[t] = sv;
    wsum += sv;
    if (lane == owner) c[slot] = -INFINITY;
  }
  if (lane == 0) {
    const float inv = (mode == 0 || norm_topk) ? 1.f / (wsum + 1e-20f) : 1.f;
    for (int t = 0; t < k; ++t) {
      idx[(size_t)row * k + t] = ik[t];
      w[(size_t)row * k + t] = wk[t] * inv * routed_scale;
    }
  }
}

__global__ __launch_bounds__(256) void moe_build_kernel(
    const int* __restrict__ idx, int* __restrict__ gather_tok,
    int* __restrict__ inv_pos, int T, int k, int E, int C) {
  __shared__ int counts[256];
  __shared__ int offsets[256];
  const int tid = threadIdx.x;
  const int A = T * k;
  for (int e = tid; e < E; e += 256) counts[e] = 0;
  __syncthreads();
  for (int a = tid; a < A; a += 256) atomicAdd(&counts[idx[a]], 1);
  __syncthreads();
  if (tid == 0) {  // E <= 256: serial prefix is ~E adds, negligible here
    int run = 0;
    for (int e = 0; e < E; ++e) {
      offsets[e] = run;
      run += counts[e];
    }
  }
  __syncthreads();
  for (int e = tid; e < E; e += 256) counts[e] = 0;  // reuse as cursors
  // default: invalid capacity slots gather token 0 (scale is 0 via inv_pos)
  for (int p = tid; p < E * C; p += 256) gather_tok[p] = 0;
  __syncthreads();
  for (int a = tid; a < A; a += 256) {
    const int e = idx[a];
    const int r = atomicAdd(&counts[e], 1);           // rank within expert
    const int global_rank = offsets[e] + r;           // dense order
    // dense position -> padded [E, C] position
    const int pos = e * C + r;                        // r < C always (count_e <= T <= C)
    gather_tok[pos] = a / k;
    inv_pos[a] = pos;
    (void)global_rank;
  }
}

// out[t, :] = sum_j w[t, j] * y[inv_pos[t*k + j], :]   (fp32 accumulate)
__global__ __launch_bounds__(256) void moe_combine_kernel(
    const unsigned short* __restrict__ y, const int* __restrict__ inv_pos,
    const float* __restrict__ w, unsigned short* __restrict__ out,
    int T, int k, int D) {
  const long long n8 = (long long)T * (D >> 3);
  const long long stride = (long long)gridDim.x * blockDim.x;
  const int d8 = D >> 3;
  for (long long i = blockIdx.x * (long long)blockDim.x + threadIdx.x; i < n8; i += stride) {
    const int t = (int)(i / d8);
    const int c8 = (int)(i % d8) * 8;
    float acc[8];
#pragma unroll
    for (int j = 0; j < 8; ++j) acc[j] = 0.f;
    for (int j = 0; j < k; ++j) {
      const float wj = w[t * k + j];
      const ushort8 v = *(const ushort8*)(y + (size_t)inv_pos[t * k + j] * D + c8);
#pragma unroll
      for (int q = 0; q < 8; ++q) acc[q] += wj * b2f(v[q]);
    }
    ushort8 o;
#pragma unroll
    for (int q = 0; q < 8; ++q) o[q] = f2b(acc[q]);
    *(ushort8*)(out + (size_t)t * D + c8) = o;
  }
}

// ---------------------------------------------------------------------------
// MLA (DeepSeek V2/V3) decode attention on matrix cores — ABSORBED form.
//
// The kv_b projection is folded into the query and output (DeepSeek's own
// inference trick): q_lat[h] = q_nope[h] @ W_k[h] lives in latent space, so
// decode attention is MQA over the cached per-token latent(512)+rope(64)
// stream — 1152 B/token TOTAL regardless of head count (the reference's
// torchtune engine cannot run MLA at all; a GQA cache for V3 would be
// n_heads*576 per token).  Per 32-position tile and 16-head group:
//   scores[16h][16p]: 18 x v_mfma_f32_16x16x32_bf16 per half-tile
//     (A = q fragments re-gathered from L1, B = 1 KB coalesced packed-cache
//      streams — same fragment geometry as the GQA kernel)
//   online softmax via 4 x shfl over 16-lane column groups (shared code shape)
//   out_lat[16h][512] += 32 x mfma (P from LDS image, V = packed latent)
// One wave per (b, head-group, split); fp32 (m, l, o[512]) partials merged
// by attn_decode_merge512.  Latent+rope cache copies are kept in the SAME
// fragment-packed layouts as the GQA kp/vp (18 qk-chunks / 32 pv-groups),
// appended by mla_append_kernel.
// ---------------------------------------------------------------------------

#define MLA_LAT 512
#define MLA_ROPE 64
#define MLA_DQK 576   // latent + rope, the absorbed q/k width
#define MLA_CHQK 18   // 32-dim MFMA chunks across DQK
#define MLA_GPV 32    // 16-dim output groups across LAT

// Fused MLA KV-side prep: raw kv_a output [B,S,576] -> RMSNorm the 512-dim
// latent (fp32 math, weight w), rope the 64-dim shared key at `positions`
// (interleaved or half convention), and write BOTH cache layouts (plain
// [B,1,T,512]/[B,1,T,64] for the eager prefill reader, fragment-packed
// kp/vp for the MFMA decode kernel). Replaces ~10 torch launches per layer
// (norm ops, rope ops, two .contiguous() copies, slice writes) with one.
// One wave per (b, s): 512 = 64 lanes x 8 for the rms reduce.
__global__ __launch_bounds__(256) void mla_prep_append_kernel(
    const unsigned short* __restrict__ ckv, const unsigned short* __restrict__ w,
    const float* __restrict__ cosb, const float* __restrict__ sinb,
    const int* __restrict__ positions,
    unsigned short* __restrict__ lat_c, unsigned short* __restrict__ rot_c,
    unsigned short* __restrict__ kp, unsigned short* __restrict__ vp,
    int B, int S, int T, int T32, float eps, int interleave, int npos,
    unsigned char* __restrict__ kp8, unsigned char* __restrict__ vp8,
    float* __restrict__ ks) {
  const int wid = blockIdx.x * (blockDim.x >> 6) + (threadIdx.x >> 6);
  if (wid >= B * S) return;
  const int lane = threadIdx.x & 63;
  const int s = wid % S;
  const int b = wid / S;
  const int pos = positions[(npos == B * S && npos != S) ? wid : s];
  const unsigned short* row = ckv + (size_t)wid * MLA_DQK;
  // ---- rms over the 512 latent dims ----
  float v[8];
  float acc = 0.f;
#pragma unroll
  for (int j = 0; j < 8; ++j) {
    v[j] = b2f(row[lane * 8 + j]);
    acc += v[j] * v[j];
  }
#pragma unroll
  for (int m = 32; m > 0; m >>= 1) acc += __shfl_xor(acc, m);
  const float inv = rsqrtf(acc / (float)MLA_LAT + eps);
  float lat[8];
#pragma unroll
  for (int j = 0; j < 8; ++j) lat[j] = v[j] * inv * b2f(w[lane * 8 + j]);
  // ---- rope the 64-dim shared key (lanes 0..31 handle one pair each) ----
  float r1 = 0.f, r2 = 0.f;
  if (lane < 32) {
    const float c = cosb[(size_t)pos * 32 + lane];
    const float sn = sinb[(size_t)pos * 32 + lane];
    int i1, i2;
    if (interleave) { i1 = lane * 2; i2 = lane * 2 + 1; }
    else            { i1 = lane;     i2 = lane + 32;    }
    const float x1 = b2f(row[MLA_LAT + i1]);
    const float x2 = b2f(row[MLA_LAT + i2]);
    // output is cat([x1c - x2s, x2c + x1s]) in HALF layout (matches _rope)
    r1 = x1 * c - x2 * sn;
    r2 = x2 * c + x1 * sn;
  }
  // plain caches (bf16, prefill reader) + bf16 packed copies
  unsigned short* lrow = lat_c + ((size_t)b * T + pos) * MLA_LAT;
  unsigned short* rrow = rot_c + ((size_t)b * T + pos) * MLA_ROPE;
  const size_t kbase = ((size_t)b * (T32 >> 4) + (pos >> 4)) * MLA_CHQK * 512;
  const size_t vbase = (size_t)b * MLA_GPV * (T32 >> 5) * 512;
#pragma unroll
  for (int j = 0; j < 8; ++j) {
    const int d = lane * 8 + j;
    lrow[d] = f2b(lat[j]);
    if (kp) {
      kp[kbase + (size_t)(d >> 5) * 512 + (((d & 31) >> 3) * 16 + (pos & 15)) * 8 + (d & 7)] = f2b(lat[j]);
      vp[vbase + ((size_t)(d >> 4) * (T32 >> 5) + (pos >> 5)) * 512
         + (((pos & 31) >> 3) * 16 + (d & 15)) * 8 + (pos & 7)] = f2b(lat[j]);
    }
  }
  if (lane < 32) {
    rrow[lane] = f2b(r1);
    rrow[lane + 32] = f2b(r2);
    if (kp) {
      const int d1 = MLA_LAT + lane, d2 = MLA_LAT + lane + 32;
      kp[kbase + (size_t)(d1 >> 5) * 512 + (((d1 & 31) >> 3) * 16 + (pos & 15)) * 8 + (d1 & 7)] = f2b(r1);
      kp[kbase + (size_t)(d2 >> 5) * 512 + (((d2 & 31) >> 3) * 16 + (pos & 15)) * 8 + (d2 & 7)] = f2b(r2);
    }
  }
  if (kp8) {
    // fp8 packed copies: one scale per token row over all 576 dims
    float mx = fmaxf(fabsf(r1), fabsf(r2));
#pragma unroll
    for (int j = 0; j < 8; ++j) mx = fmaxf(mx, fabsf(lat[j]));
#pragma unroll
    for (int m = 32; m > 0; m >>= 1) mx = fmaxf(mx, __shfl_xor(mx, m));
    const float scl = fmaxf(mx, 1e-12f) / 448.f;
    const float qinv = 1.f / scl;
    if (lane == 0) ks[(size_t)b * T32 + pos] = scl;
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      const int d = lane * 8 + j;
      const unsigned short pk = (unsigned short)__builtin_amdgcn_cvt_pk_fp8_f32(lat[j] * qinv, 0.f, 0, false);
      kp8[kbase + (size_t)(d >> 5) * 512 + (((d & 31) >> 3) * 16 + (pos & 15)) * 8 + (d & 7)] = (unsigned char)(pk & 0xff);
      vp8[vbase + ((size_t)(d >> 4) * (T32 >> 5) + (pos >> 5)) * 512
          + (((pos & 31) >> 3) * 16 + (d & 15)) * 8 + (pos & 7)] = (unsigned char)(pk & 0xff);
    }
    if (lane < 32) {
      const int d1 = MLA_LAT + lane, d2 = MLA_LAT + lane + 32;
      const unsigned short p1 = (unsigned short)__builtin_amdgcn_cvt_pk_fp8_f32(r1 * qinv, 0.f, 0, false);
      const unsigned short p2 = (unsigned short)__builtin_amdgcn_cvt_pk_fp8_f32(r2 * qinv, 0.f, 0, false);
      kp8[kbase + (size_t)(d1 >> 5) * 512 + (((d1 & 31) >> 3) * 16 + (pos & 15)) * 8 + (d1 & 7)] = (unsigned char)(p1 & 0xff);
      kp8[kbase + (size_t)(d2 >> 5) * 512 + (((d2 & 31) >> 3) * 16 + (pos & 15)) * 8 + (d2 & 7)] = (unsigned char)(p2 & 0xff);
    }
  }
}

// q-side finisher: rope the 64-dim query tail and assemble the absorbed
// query [B, H, 576] = [q_lat(512) | rope(q_rot)(64)] in one launch
// (replaces ~6 torch ops per layer: rope mul/cat x2, cat, contiguous).
// One wave per (b, h): q strided [B, S=1, H, 192], q_lat [B, 1, H, 512].
__global__ __launch_bounds__(256) void mla_q_prep_kernel(
    const unsigned short* __restrict__ q, const unsigned short* __restrict__ q_lat,
    const float* __restrict__ cosb, const float* __restrict__ sinb,
    const int* __restrict__ positions, unsigned short* __restrict__ qfull,
    int B, int H, long long q_bstride, int nope, int interleave, int npos,
    unsigned char* __restrict__ q8, float* __restrict__ sq) {
  const int wid = blockIdx.x * (blockDim.x >> 6) + (threadIdx.x >> 6);
  if (wid >= B * H) return;
  const int lane = threadIdx.x & 63;
  const int h = wid % H;
  const int b = wid / H;
  const unsigned short* lsrc = q_lat + ((size_t)b * H + h) * MLA_LAT;
  float lv[8];
#pragma unroll
  for (int j = 0; j < 8; ++j) lv[j] = b2f(lsrc[lane * 8 + j]);
  float r1 = 0.f, r2 = 0.f;
  if (lane < 32) {
    const int pos = positions[(npos == B) ? b : 0];
    const float c = cosb[(size_t)pos * 32 + lane];
    const float sn = sinb[(size_t)pos * 32 + lane];
    const unsigned short* qrot = q + (size_t)b * q_bstride + (size_t)h * (nope + MLA_ROPE) + nope;
    int i1, i2;
    if (interleave) { i1 = lane * 2; i2 = lane * 2 + 1; }
    else            { i1 = lane;     i2 = lane + 32;    }
    const float x1 = b2f(qrot[i1]);
    const float x2 = b2f(qrot[i2]);
    r1 = x1 * c - x2 * sn;
    r2 = x2 * c + x1 * sn;
  }
  if (q8 == nullptr) {
    unsigned short* dst = qfull + ((size_t)b * H + h) * MLA_DQK;
#pragma unroll
    for (int j = 0; j < 8; ++j) dst[lane * 8 + j] = f2b(lv[j]);
    if (lane < 32) {
      dst[MLA_LAT + lane] = f2b(r1);
      dst[MLA_LAT + lane + 32] = f2b(r2);
    }
    return;
  }
  // fp8 output: one e4m3 scale per (b, h) query row over all 576 dims
  float mx = fmaxf(fabsf(r1), fabsf(r2));
#pragma unroll
  for (int j = 0; j < 8; ++j) mx = fmaxf(mx, fabsf(lv[j]));
#pragma unroll
  for (int m = 32; m > 0; m >>= 1) mx = fmaxf(mx, __shfl_xor(mx, m));
  const float scl = fmaxf(mx, 1e-12f) / 448.f;
  const float inv = 1.f / scl;
  if (lane == 0) sq[(size_t)b * H + h] = scl;
  unsigned char* dst8 = q8 + ((size_t)b * H + h) * MLA_DQK;
#pragma unroll
  for (int j = 0; j < 8; ++j) {
    const unsigned short pk = (unsigned short)__builtin_amdgcn_cvt_pk_fp8_f32(lv[j] * inv, 0.f, 0, false);
    dst8[lane * 8 + j] = (unsigned char)(pk & 0xff);
  }
  if (lane < 32) {
    const unsigned short p1 = (unsigned short)__builtin_amdgcn_cvt_pk_fp8_f32(r1 * inv, 0.f, 0, false);
    const unsigned short p2 = (unsigned short)__builtin_amdgcn_cvt_pk_fp8_f32(r2 * inv, 0.f, 0, false);
    dst8[MLA_LAT + lane] = (unsigned char)(p1 & 0xff);
    dst8[MLA_LAT + lane + 32] = (unsigned char)(p2 & 0xff);
  }
}

__global__ __launch_bounds__(256) void mla_append_kernel(
    const unsigned short* __restrict__ lat, const unsigned short* __restrict__ rot,
    const int* __restrict__ positions, unsigned short* __restrict__ kp,
    unsigned short* __restrict__ vp, int B, int S, int T32, int npos) {
  // wave per (b, s); lane covers dims d = lane*9 .. lane*9+8 (576 = 64*9)
  const int wid = blockIdx.x * (blockDim.x >> 6) + (threadIdx.x >> 6);
  if (wid >= B * S) return;
  const int lane = threadIdx.x & 63;
  const int s = wid % S;
  const int b = wid / S;
  const int pos = positions[(npos == B * S && npos != S) ? wid : s];
  const unsigned short* lrow = lat + ((size_t)b * S + s) * MLA_LAT;
  const unsigned short* rrow = rot + ((size_t)b * S + s) * MLA_ROPE;
  const size_t kbase = (size_t)b * (T32 >> 4) * MLA_CHQK * 512 + (size_t)(pos >> 4) * MLA_CHQK * 512;
  const size_t vbase = (size_t)b * MLA_GPV * (T32 >> 5) * 512;
#pragma unroll
  for (int i = 0; i < 9; ++i) {
    const int d = lane * 9 + i;
    const unsigned short v = (d < MLA_LAT) ? lrow[d] : rrow[d - MLA_LAT];
    // K-fragment image (16 pos x 32 dims per chunk)
    kp[kbase + (size_t)(d >> 5) * 512 + (((d & 31) >> 3) * 16 + (pos & 15)) * 8 + (d & 7)] = v;
    if (d < MLA_LAT) {
      // V-fragment image (32 pos x 16 dims per group)
      vp[vbase + ((size_t)(d >> 4) * (T32 >> 5) + (pos >> 5)) * 512
         + (((pos & 31) >> 3) * 16 + (d & 15)) * 8 + (pos & 7)] = v;
    }
  }
}

template <bool FP8 = false>
__global__ __launch_bounds__(256) void attn_decode_mla_kernel(
    const unsigned short* __restrict__ q, const unsigned short* __restrict__ kp,
    const unsigned short* __restrict__ vp, const int* __restrict__ seq_lens,
    float* __restrict__ ws_o, float* __restrict__ ws_ml,
    int B, int H, int T32, int nsplit, float scale,
    const float* __restrict__ sq = nullptr, const float* __restrict__ ks = nullptr) {
  const int wv = threadIdx.x >> 6;
  const int wid = blockIdx.x * 4 + wv;
  const int hgroups = (H + 15) >> 4;
  __shared__ unsigned short plds_all[4][16 * 48];
  if (wid >= B * hgroups * nsplit) return;
  const int split = wid % nsplit;
  const int hg = (wid / nsplit) % hgroups;
  const int b = wid / (nsplit * hgroups);
  const int lane = threadIdx.x & 63;
  const int sl = seq_lens[b];
  const int chunk = ((T32 / nsplit + 31) >> 5) << 5;
  const int c0 = split * chunk;
  const int c1 = min(c0 + chunk, sl);
  unsigned short* plds = plds_all[wv];

  const int nq = min(16, H - hg * 16);
  const int qi = min(lane & 15, nq - 1);
  const unsigned short* qrow = q + ((size_t)b * H + hg * 16 + qi) * MLA_DQK + (lane >> 4) * 8;
  const unsigned char* qrow8 = reinterpret_cast<const unsigned char*>(q)
      + ((size_t)b * H + hg * 16 + qi) * MLA_DQK + (lane >> 4) * 8;
  const unsigned char* kp8 = reinterpret_cast<const unsigned char*>(kp);
  const unsigned char* vp8 = reinterpret_cast<const unsigned char*>(vp);
  float srow[4], Rscale = 1.f;
  if (FP8) {
    const float sqv = sq[(size_t)b * H + hg * 16 + qi];
#pragma unroll
    for (int r = 0; r < 4; ++r) srow[r] = __shfl(sqv, (lane >> 4) * 4 + r);
  }

  float m[4], lsum[4];
#pragma unroll
  for (int r = 0; r < 4; ++r) { m[r] = -INFINITY; lsum[r] = 0.f; }
  floatx4 acco[MLA_GPV];
#pragma unroll
  for (int g = 0; g < MLA_GPV; ++g) acco[g] = (floatx4)(0.f);

  const size_t kbase = (size_t)b * (T32 >> 4) * MLA_CHQK * 512;
  const size_t vbase = (size_t)b * MLA_GPV * (T32 >> 5) * 512;
  const int col = lane & 15;

  for (int t = c0; t < c1; t += 32) {
    floatx4 sc[2];
#pragma unroll
    for (int h = 0; h < 2; ++h) sc[h] = (floatx4)(0.f);
    // scores over the 18 qk chunks; q fragments re-gathered per chunk
    // (L1-resident after the first tile), k streamed packed
    for (int c = 0; c < MLA_CHQK; ++c) {
      if (FP8) {
        const long a = *reinterpret_cast<const long*>(qrow8 + c * 32);
#pragma unroll
        for (int h = 0; h < 2; ++h) {
          const unsigned char* kt = kp8 + kbase
              + ((size_t)((t >> 4) + h) * MLA_CHQK + c) * 512 + (size_t)lane * 8;
          const long kb = __builtin_nontemporal_load(reinterpret_cast<const long*>(kt));
          sc[h] = __builtin_amdgcn_mfma_f32_16x16x32_fp8_fp8(a, kb, sc[h], 0, 0, 0);
        }
      } else {
        const bf16x8 a = *reinterpret_cast<const bf16x8*>(qrow + c * 32);
#pragma unroll
        for (int h = 0; h < 2; ++h) {
          const unsigned short* kt = kp + kbase
              + ((size_t)((t >> 4) + h) * MLA_CHQK + c) * 512 + (size_t)lane * 8;
          const bf16x8 kb = __builtin_nontemporal_load(reinterpret_cast<const bf16x8*>(kt));
          sc[h] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, kb, sc[h], 0, 0, 0);
        }
      }
    }
    float rmax[4];
#pragma unroll
    for (int h = 0; h < 2; ++h) {
      const int pos = t + h * 16 + col;
      const bool ok = pos < c1;
      const float skc = FP8 ? ks[(size_t)b * T32 + min(pos, T32 - 1)] : 1.f;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        float sv_ = sc[h][r] * scale;
        if (FP8) sv_ *= srow[r] * skc;
        sc[h][r] = ok ? sv_ : -INFINITY;
      }
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) rmax[r] = fmaxf(sc[0][r], sc[1][r]);
#pragma unroll
    for (int mm = 1; mm < 16; mm <<= 1)
#pragma unroll
      for (int r = 0; r < 4; ++r) rmax[r] = fmaxf(rmax[r], __shfl_xor(rmax[r], mm));
    float alpha[4], rsum[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const float mn = fmaxf(m[r], rmax[r]);
      alpha[r] = (lsum[r] > 0.f) ? __expf(m[r] - mn) : 0.f;
      m[r] = mn;
      const float p0 = __expf(sc[0][r] - mn);
      const float p1 = __expf(sc[1][r] - mn);
      sc[0][r] = p0;
      sc[1][r] = p1;
      rsum[r] = p0 + p1;
    }
#pragma unroll
    for (int mm = 1; mm < 16; mm <<= 1)
#pragma unroll
      for (int r = 0; r < 4; ++r) rsum[r] += __shfl_xor(rsum[r], mm);
#pragma unroll
    for (int r = 0; r < 4; ++r) lsum[r] = lsum[r] * alpha[r] + rsum[r];
    float s_pv = 1.f, rfac = 1.f;
    if (FP8) {
      float mv = ks[(size_t)b * T32 + min(t + (lane & 31), T32 - 1)];
#pragma unroll
      for (int m_ = 32; m_ > 0; m_ >>= 1) mv = fmaxf(mv, __shfl_xor(mv, m_));
      s_pv = fmaxf(mv, 1e-12f);
      rfac = Rscale / s_pv;
      Rscale = s_pv;
    }
#pragma unroll
    for (int g = 0; g < MLA_GPV; ++g)
#pragma unroll
      for (int r = 0; r < 4; ++r) acco[g][r] *= alpha[r] * (FP8 ? rfac : 1.f);
    long pf8 = 0;
    bf16x8 pf;
    if (FP8) {
      unsigned char* pl8 = reinterpret_cast<unsigned char*>(plds);
#pragma unroll
      for (int h = 0; h < 2; ++h) {
        const int pos = t + h * 16 + col;
        const float svv = ks[(size_t)b * T32 + min(pos, T32 - 1)];
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const unsigned short pk = (unsigned short)__builtin_amdgcn_cvt_pk_fp8_f32(
              sc[h][r] * svv / s_pv, 0.f, 0, false);
          pl8[((lane >> 4) * 4 + r) * 48 + h * 16 + col] = (unsigned char)(pk & 0xff);
        }
      }
      pf8 = *reinterpret_cast<const long*>(pl8 + (lane & 15) * 48 + (lane >> 4) * 8);
      const unsigned char* vt8 = vp8 + vbase + (size_t)(t >> 5) * 512 + (size_t)lane * 8;
      for (int g = 0; g < MLA_GPV; ++g) {
        const long vb = __builtin_nontemporal_load(
            reinterpret_cast<const long*>(vt8 + (size_t)g * (T32 >> 5) * 512));
        acco[g] = __builtin_amdgcn_mfma_f32_16x16x32_fp8_fp8(pf8, vb, acco[g], 0, 0, 0);
      }
    } else {
#pragma unroll
      for (int h = 0; h < 2; ++h)
#pragma unroll
        for (int r = 0; r < 4; ++r)
          plds[((lane >> 4) * 4 + r) * 48 + h * 16 + col] = f2b(sc[h][r]);
      pf = *reinterpret_cast<const bf16x8*>(plds + (lane & 15) * 48 + (lane >> 4) * 8);
      const unsigned short* vt = vp + vbase + (size_t)(t >> 5) * 512 + (size_t)lane * 8;
      for (int g = 0; g < MLA_GPV; ++g) {
        const bf16x8 vb = __builtin_nontemporal_load(
            reinterpret_cast<const bf16x8*>(vt + (size_t)g * (T32 >> 5) * 512));
        acco[g] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(pf, vb, acco[g], 0, 0, 0);
      }
    }
  }

#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int qrow_i = (lane >> 4) * 4 + r;
    if (qrow_i < nq) {
      const size_t pidx = ((size_t)(b * H + hg * 16 + qrow_i) * nsplit + split);
      for (int g = 0; g < MLA_GPV; ++g)
        ws_o[pidx * MLA_LAT + g * 16 + col] = acco[g][r] * (FP8 ? Rscale : 1.f);
      if (col == 0) {
        ws_ml[pidx * 2 + 0] = m[r];
        ws_ml[pidx * 2 + 1] = lsum[r];
      }
    }
  }
}

// wide merge for the MLA 512-dim latent output: 256 threads, 2 dims each
__global__ __launch_bounds__(256) void attn_decode_merge512(
    const float* __restrict__ ws_o, const float* __restrict__ ws_ml,
    unsigned short* __restrict__ out, int nsplit) {
  const int bh = blockIdx.x;
  float M = -INFINITY;
  for (int i = 0; i < nsplit; ++i) M = fmaxf(M, ws_ml[((size_t)bh * nsplit + i) * 2 + 0]);
#pragma unroll
  for (int e = 0; e < 2; ++e) {
    const int d = threadIdx.x + e * 256;
    float L = 0.f, O = 0.f;
    for (int i = 0; i < nsplit; ++i) {
      const float lg = ws_ml[((size_t)bh * nsplit + i) * 2 + 1];
      const float alpha = (lg > 0.f) ? __expf(ws_ml[((size_t)bh * nsplit + i) * 2 + 0] - M) : 0.f;
      L += alpha * lg;
      O += alpha * ws_o[((size_t)bh * nsplit + i) * MLA_LAT + d];
    }
    out[(size_t)bh * MLA_LAT + d] = f2b(L > 0.f ? O / L : 0.f);
  }
}

// ---------------------------------------------------------------------------
// SwiGLU: silu(gate) * up, elementwise, vectorized
// ---------------------------------------------------------------------------

__global__ __launch_bounds__(256) void swiglu_kernel(
    const unsigned short* __restrict__ g, const unsigned short* __restrict__ u,
    unsigned short* __restrict__ out, long long n8) {
  const long long stride = (long long)gridDim.x * blockDim.x;
  for (long long i = blockIdx.x * (long long)blockDim.x + threadIdx.x; i < n8; i += stride) {
    ushort8 gv = *(const ushort8*)(g + i * 8);
    ushort8 uv = *(const ushort8*)(u + i * 8);
    ushort8 o;
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      const float gf = b2f(gv[j]);
      const float s = gf * __builtin_amdgcn_rcpf(1.f + __expf(-gf));
      o[j] = f2b(s * b2f(uv[j]));
    }
    *(ushort8*)(out + i * 8) = o;
  }
}

// packed variant: gu = [rows, 2*I] from the fused gate_up GEMM ([gate | up])
__global__ __launch_bounds__(256) void swiglu_packed_kernel(
    const unsigned short* __restrict__ gu, unsigned short* __restrict__ out,
    long long rows, int I) {
  const long long n8 = rows * (I >> 3);
  const long long stride = (long long)gridDim.x * blockDim.x;
  const int i8 = I >> 3;
  for (long long i = blockIdx.x * (long long)blockDim.x + threadIdx.x; i < n8; i += stride) {
    const long long row = i / i8;
    const long long col8 = i % i8;
    const unsigned short* base = gu + row * (2LL * I) + col8 * 8;
    ushort8 gv = *(const ushort8*)base;
    ushort8 uv = *(const ushort8*)(base + I);
    ushort8 o;
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      const float gf = b2f(gv[j]);
      const float s = gf * __builtin_amdgcn_rcpf(1.f + __expf(-gf));
      o[j] = f2b(s * b2f(uv[j]));
    }
    *(ushort8*)(out + i * 8) = o;
  }
}

// packed GeGLU (gemma2): gelu_tanh(gate) * up on the fused [gate | up] GEMM
// output — same stream shape as swiglu_packed, tanh-approximate gelu in fp32.
__global__ __launch_bounds__(256) void geglu_packed_kernel(
    const unsigned short* __restrict__ gu, unsigned short* __restrict__ out,
    long long rows, int I) {
  const long long n8 = rows * (I >> 3);
  const long long stride = (long long)gridDim.x * blockDim.x;
  const int i8 = I >> 3;
  for (long long i = blockIdx.x * (long long)blockDim.x + threadIdx.x; i < n8; i += stride) {
    const long long row = i / i8;
    const long long col8 = i % i8;
    const unsigned short* base = gu + row * (2LL * I) + col8 * 8;
    ushort8 gv = *(const ushort8*)base;
    ushort8 uv = *(const ushort8*)(base + I);
    ushort8 o;
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      const float gf = b2f(gv[j]);
      const float g3 = 0.7978845608028654f * (gf + 0.044715f * gf * gf * gf);
      const float s = 0.5f * gf * (1.f + tanhf(g3));
      o[j] = f2b(s * b2f(uv[j]));
    }
    *(ushort8*)(out + i * 8) = o;
  }
}

// ---------------------------------------------------------------------------
// Skinny decode GEMM: Y[M,N] = X[M,K] @ W[N,K]^T, bf16, M <= 256 (decode
// batch).  This is the decode hot path's dominant cost (the reference runs
// every projection through torchtune's nn.Linear -> cuBLAS,
// llm_utils.py:491-500 / general_mha.py:83-102); at decode shapes the GEMM is
// pure weight streaming and hipBLASLt leaves bandwidth on the table at large
// K (down_proj [M,28672]x[28672,8192] measured 3.6 TB/s vs ~6.3 achievable).
//
// Design (MI355X / CDNA4):
//   * computed as D^T = W . X^T on v_mfma_f32_32x32x16_bf16: the A operand
//     (W, the streamed 0.1-2 GB operand) and the B operand (X, L2/L3
//     resident) are BOTH k-contiguous 16 B per lane in this orientation, so
//     no transpose and no LDS staging at all -- per the CDNA4 guide's
//     "GEMV / small-M decode weights: load straight to VGPRs, deep unroll,
//     late vmcnt" rule.  Each 128 B cache line of W is consumed by 8
//     fragment loads of the same wave (L1-absorbed).
//   * grid = (N/BN) * SPLITK workgroups of 4 waves; BN = 128 (one 32-row
//     n-tile per wave); SPLITK chosen so the grid oversubscribes the 256 CUs
//     (>= 2 blocks/CU) while K/SPLITK stays >= ~1024 (latency amortized).
//   * fp32 split-K partials + a tiny vectorized combine kernel (bias fused);
//     SPLITK == 1 writes bf16 directly.
// ---------------------------------------------------------------------------

DEVINL bf16x8 load_bf16x8(const unsigned short* p) {
  return *reinterpret_cast<const bf16x8*>(p);
}

// MT = M/32 (1..8). One workgroup computes Y[0:M, n0:n0+128] over k-range
// [k0, k1). Lane l of wave w holds A row (n0 + w*32 + (l&31)), k-chunk
// (l>>5)*8; B col (mt*32 + (l&31)) of X with the same k-chunk.
template <int MT, bool SPLIT>
__global__ __launch_bounds__(256) void skinny_gemm_kernel(
    const unsigned short* __restrict__ W, const unsigned short* __restrict__ X,
    unsigned short* __restrict__ Y, float* __restrict__ P,
    const unsigned short* __restrict__ bias,
    int N, long long K, int kc, int nsplit) {
  const int ntiles = N >> 7;
  const int tile = blockIdx.x % ntiles;
  const int split = blockIdx.x / ntiles;
  const long long k0 = (long long)split * kc;
  const long long k1 = min(k0 + (long long)kc, K);
  const int lane = threadIdx.x & 63;
  const int wv = threadIdx.x >> 6;
  const int n0 = tile * 128 + wv * 32;
  const int arow = n0 + (lane & 31);
  const long long koff = (lane >> 5) * 8;

  floatx16 acc[MT];
#pragma unroll
  for (int t = 0; t < MT; ++t) acc[t] = (floatx16)(0.f);

  const unsigned short* wp = W + (size_t)arow * K + k0 + koff;
  const unsigned short* xp = X + (size_t)(lane & 31) * K + k0 + koff;

  long long k = k0;
#pragma unroll 1
  for (; k + 64 <= k1; k += 64) {
    bf16x8 a[4], b[4][MT];
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      a[u] = load_bf16x8(wp + u * 16);
#pragma unroll
      for (int t = 0; t < MT; ++t) b[u][t] = load_bf16x8(xp + (size_t)t * 32 * K + u * 16);
    }
#pragma unroll
    for (int u = 0; u < 4; ++u)
#pragma unroll
      for (int t = 0; t < MT; ++t)
        acc[t] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(a[u], b[u][t], acc[t], 0, 0, 0);
    wp += 64;
    xp += 64;
  }
  for (; k < k1; k += 16) {
    bf16x8 a = load_bf16x8(wp);
#pragma unroll
    for (int t = 0; t < MT; ++t) {
      bf16x8 b = load_bf16x8(xp + (size_t)t * 32 * K);
      acc[t] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(a, b, acc[t], 0, 0, 0);
    }
    wp += 16;
    xp += 16;
  }

  // D layout (32x32): m = lane&31 (col), n_local = (r&3) + 8*(r>>2) + 4*(lane>>5)
  const int m_local = lane & 31;
  const int nbase = n0 + 4 * (lane >> 5);
#pragma unroll
  for (int t = 0; t < MT; ++t) {
    const int m = t * 32 + m_local;
    if (SPLIT) {
      float* prow = P + ((size_t)split * (MT * 32) + m) * N;  // P layout [nsplit, M, N]
#pragma unroll
      for (int g = 0; g < 4; ++g) {
        floatx4 v4;
#pragma unroll
        for (int j = 0; j < 4; ++j) v4[j] = acc[t][g * 4 + j];
        *reinterpret_cast<floatx4*>(prow + nbase + g * 8) = v4;
      }
    } else {
      unsigned short* yrow = Y + (size_t)m * N;
#pragma unroll
      for (int g = 0; g < 4; ++g) {
        unsigned short o[4];
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          float v = acc[t][g * 4 + j];
          if (bias) v += b2f(bias[nbase + g * 8 + j]);
          o[j] = f2b(v);
        }
        *reinterpret_cast<unsigned long long*>(yrow + nbase + g * 8) =
            *reinterpret_cast<unsigned long long*>(o);
      }
    }
  }
}

// ---------------------------------------------------------------------------
// v2: prepacked-weight variant.  W is pre-shuffled ONCE at load time into
// MFMA A-fragment order: [N/32][K/16][lane 0..63][8 bf16], lane = (k-half)*32
// + n-row — so each A-fragment load is one fully-coalesced wave-wide 1 KB
// stream (v1's fragment-shaped 16 B gathers are TA/load-path-bound: measured
// 2.0 vs 5.3 TB/s).  X is staged cooperatively per 64-k step into a padded
// LDS image (row stride 72 elems = 144 B -> ds_read_b128 bank-conflict-free)
// and read back as B fragments.  K % 64 == 0 required.
// ---------------------------------------------------------------------------

// Also the MoE grouped-GEMM kernel (the reference's latent
// MOEExpert/MOELayer scaffolding, llm_utils.py:502-590, never executed): for
// Mixtral-class decode each expert e (blockIdx.y) computes its own
// [C, N] = [C, K] @ Wp_e^T over a fixed per-expert token capacity C — one
// launch covers every expert, weights stream from the stacked prepack.
template <int MT, bool SPLIT, int BK, bool SWIGLU = false>
__global__ __launch_bounds__(256) void skinny_gemm_packed_kernel(
    const unsigned short* __restrict__ Wp, const unsigned short* __restrict__ X,
    unsigned short* __restrict__ Y, float* __restrict__ P,
    const unsigned short* __restrict__ bias,
    int N, long long K, int kc, int nsplit, long long ldx = 0) {
  // SWIGLU: X is the fused [rows, 2K] gate|up GEMM output; the staging
  // computes silu(gate)*up on the fly (row stride ldx = 2K, up at +K) —
  // the intermediate activation tensor never exists (saves its write +
  // read, ~29 MB/layer at 70B B=128, and one launch per layer).
  if (!SWIGLU) ldx = K;
  constexpr int BKC = BK / 16;   // MFMA k-chunks (A fragments) per K-step
  constexpr int XROW = BK + 8;   // padded LDS row stride (elems): conflict-free b128
  const int ntiles = N >> 7;
  const int tile = blockIdx.x % ntiles;
  const int split = blockIdx.x / ntiles;
  // grouped mode: expert blockIdx.y owns rows [e*MT*32, (e+1)*MT*32) of X/Y
  // and its own weight block; gridDim.y == 1 degenerates to the plain GEMM.
  const int e = blockIdx.y;
  Wp += (size_t)e * (size_t)N * (size_t)K;
  X += (size_t)e * (size_t)(MT * 32) * (size_t)K;
  const long long k0 = (long long)split * kc;
  const long long k1 = min(k0 + (long long)kc, K);
  if (k0 >= k1) return;
  const int lane = threadIdx.x & 63;
  const int wv = threadIdx.x >> 6;
  const int tid = threadIdx.x;

  __shared__ unsigned short xs[MT * 32 * XROW];

  floatx16 acc[MT];
#pragma unroll
  for (int t = 0; t < MT; ++t) acc[t] = (floatx16)(0.f);

  // A stream: packed row for this wave's 32-n tile
  const int n32 = tile * 4 + wv;
  const unsigned short* wp = Wp + ((size_t)n32 * (K >> 4) + (k0 >> 4)) * 512 + (size_t)lane * 8;
  // X stage: thread tid covers 16 B pieces p = tid + i*256 (coalesced);
  // row = p / (BK/8), piece-in-row q = p % (BK/8); global [M, K] row-major.
  constexpr int PPT = MT * BK / 64;  // pieces per thread per step
  const int nsteps = (int)((k1 - k0) >> (BK == 64 ? 6 : 7));
  ushort8 xv[PPT];
  bf16x8 a_buf[2][BKC];
  // per-thread staging base + uniform per-piece offsets: piece p = tid+i*256
  // has row = tid/(BK/8) + i*ROWS_PER_I and column-piece q = tid%(BK/8), so
  // one VGPR pointer plus SGPR/immediate strides replaces the old per-piece
  // pointer arrays (saves ~10 VGPRs -> a wave/SIMD at MT=4)
  constexpr int ROWS_PER_I = 2048 / BK;  // rows advanced per i (256 threads)
  const unsigned short* xpb = X + k0 + (size_t)(tid / (BK / 8)) * ldx + (tid % (BK / 8)) * 8;
  const int xsb = (tid / (BK / 8)) * XROW + (tid % (BK / 8)) * 8;
  const long long xstride_i = (long long)ROWS_PER_I * ldx;

  // prologue: stage step 0, preload A(0) and A(1).  The W stream is read
  // exactly once per launch -> non-temporal (L1-bypass) loads; depth-2
  // prefetch keeps 2*BK*32n*2B per wave in flight across staging barriers.
  const unsigned short* wp1 = (nsteps > 1) ? wp + BKC * 512 : wp;  // clamp: no OOB at nsteps==1
#pragma unroll
  for (int i = 0; i < PPT; ++i) {
    xv[i] = *(const ushort8*)(xpb + i * xstride_i);
    if (SWIGLU) {
      const ushort8 up = *(const ushort8*)(xpb + i * xstride_i + K);
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        const float g = b2f(xv[i][j]);
        xv[i][j] = f2b(g * __builtin_amdgcn_rcpf(1.f + __expf(-g)) * b2f(up[j]));
      }
    }
  }
#pragma unroll
  for (int u = 0; u < BKC; ++u) {
    a_buf[0][u] = __builtin_nontemporal_load(reinterpret_cast<const bf16x8*>(wp + u * 512));
    a_buf[1][u] = __builtin_nontemporal_load(reinterpret_cast<const bf16x8*>(wp1 + u * 512));
  }
  wp += 2 * BKC * 512;
#pragma unroll
  for (int i = 0; i < PPT; ++i) *(ushort8*)(xs + xsb + i * ROWS_PER_I * XROW) = xv[i];
  __syncthreads();

  // NOTE: the A double-buffer index must be a compile-time constant — a
  // dynamic a_buf[s & 1] spills the whole array to scratch (measured 25-40x).
#define SGP_STEP(BUF)                                                                          \
  {                                                                                            \
    const bool last = (s == nsteps - 1);                                                       \
    if (!last) {                                                                               \
      _Pragma("unroll")                                                                        \
      for (int i = 0; i < PPT; ++i) {                                                          \
        xv[i] = *(const ushort8*)(xpb + i * xstride_i + (size_t)(s + 1) * BK);                 \
        if (SWIGLU) {                                                                          \
          const ushort8 up_ = *(const ushort8*)(xpb + i * xstride_i + (size_t)(s + 1) * BK + K); \
          _Pragma("unroll")                                                                    \
          for (int j_ = 0; j_ < 8; ++j_) {                                                     \
            const float g_ = b2f(xv[i][j_]);                                                   \
            xv[i][j_] = f2b(g_ * __builtin_amdgcn_rcpf(1.f + __expf(-g_)) * b2f(up_[j_]));     \
          }                                                                                    \
        }                                                                                      \
      }                                                                                        \
    }                                                                                          \
    _Pragma("unroll")                                                                          \
    for (int u = 0; u < BKC; ++u) {                                                            \
      _Pragma("unroll")                                                                        \
      for (int t = 0; t < MT; ++t) {                                                           \
        const bf16x8 b = *reinterpret_cast<const bf16x8*>(                                     \
            xs + t * 32 * XROW + (lane & 31) * XROW + u * 16 + (lane >> 5) * 8);               \
        acc[t] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(a_buf[BUF][u], b, acc[t], 0, 0, 0);   \
      }                                                                                        \
    }                                                                                          \
    if (s + 2 < nsteps) {                                                                      \
      _Pragma("unroll")                                                                        \
      for (int u = 0; u < BKC; ++u)                                                            \
        a_buf[BUF][u] = __builtin_nontemporal_load(reinterpret_cast<const bf16x8*>(wp + u * 512)); \
      wp += BKC * 512;                                                                         \
    }                                                                                          \
    if (!last) {                                                                               \
      __syncthreads();                                                                         \
      _Pragma("unroll")                                                                        \
      for (int i = 0; i < PPT; ++i) *(ushort8*)(xs + xsb + i * ROWS_PER_I * XROW) = xv[i];     \
      __syncthreads();                                                                         \
    }                                                                                          \
  }

  int s = 0;
  while (s + 2 <= nsteps) {
    SGP_STEP(0);
    ++s;
    SGP_STEP(1);
    ++s;
  }
  if (s < nsteps) SGP_STEP(0);
#undef SGP_STEP

  const int m_local = lane & 31;
  const int rows_total = gridDim.y * MT * 32;  // across all experts
  const int nbase = tile * 128 + wv * 32 + 4 * (lane >> 5);
#pragma unroll
  for (int t = 0; t < MT; ++t) {
    const int m = e * MT * 32 + t * 32 + m_local;
    if (SPLIT) {
      float* prow = P + ((size_t)split * rows_total + m) * N;
#pragma unroll
      for (int g = 0; g < 4; ++g) {
        floatx4 v4;
#pragma unroll
        for (int j = 0; j < 4; ++j) v4[j] = acc[t][g * 4 + j];
        *reinterpret_cast<floatx4*>(prow + nbase + g * 8) = v4;
      }
    } else {
      unsigned short* yrow = Y + (size_t)m * N;
#pragma unroll
      for (int g = 0; g < 4; ++g) {
        unsigned short o[4];
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          float v = acc[t][g * 4 + j];
          if (bias) v += b2f(bias[nbase + g * 8 + j]);
          o[j] = f2b(v);
        }
        *reinterpret_cast<unsigned long long*>(yrow + nbase + g * 8) =
            *reinterpret_cast<unsigned long long*>(o);
      }
    }
  }
}

// ---------------------------------------------------------------------------
// v3: packed-A + register-resident-X variant for the M=128/256 decode shapes.
// The LDS-staged v2 wins at M<=64, but at MT>=4 its X staging doubles
// (16 KB/step), the barrier pairs serialize the A stream, and the staging
// registers push the allocation to 156+ VGPRs (3 waves/SIMD).  Here X is
// never staged: each lane loads its B fragments straight from global
// (16 B per lane, same pattern as v1's B path).  X is tiny (M x K bf16,
// 2-4 MB) and every n-tile re-reads it, so after the first touch the
// fragments come from L2/L3, not HBM -- the gather that made v1's A path
// 2.0 TB/s is harmless on the B side.  No LDS, no barriers; A keeps v2's
// coalesced non-temporal 1 KB wave streams with depth-2 step prefetch.
// B chunks are loaded just-in-time per 16-k chunk (bb[MT] live registers):
// at MT=4 the allocation stays ~128 VGPRs = 4 waves/SIMD, and the vmcnt
// wait on one chunk's L2 hit is covered by the other waves' MFMA clusters.
// ---------------------------------------------------------------------------
template <int MT, bool SPLIT>
__global__ __launch_bounds__(256) void skinny_gemm_packed_xreg_kernel(
    const unsigned short* __restrict__ Wp, const unsigned short* __restrict__ X,
    unsigned short* __restrict__ Y, float* __restrict__ P,
    const unsigned short* __restrict__ bias,
    int N, long long K, int kc, int nsplit) {
  const int ntiles = N >> 7;
  const int tile = blockIdx.x % ntiles;
  const int split = blockIdx.x / ntiles;
  const int e = blockIdx.y;  // grouped mode (gridDim.y == 1 for plain GEMM)
  Wp += (size_t)e * (size_t)N * (size_t)K;
  X += (size_t)e * (size_t)(MT * 32) * (size_t)K;
  const long long k0 = (long long)split * kc;
  const long long k1 = min(k0 + (long long)kc, K);
  if (k0 >= k1) return;
  const int lane = threadIdx.x & 63;
  const int wv = threadIdx.x >> 6;
  const int n32 = tile * 4 + wv;

  const unsigned short* wp = Wp + ((size_t)n32 * (K >> 4) + (k0 >> 4)) * 512 + (size_t)lane * 8;
  // B fragment base per m-tile: row (t*32 + lane&31), k-half (lane>>5)*8
  const unsigned short* xt[MT];
#pragma unroll
  for (int t = 0; t < MT; ++t)
    xt[t] = X + (size_t)(t * 32 + (lane & 31)) * K + k0 + ((lane >> 5) * 8);

  floatx16 acc[MT];
#pragma unroll
  for (int t = 0; t < MT; ++t) acc[t] = (floatx16)(0.f);

  const int nsteps = (int)((k1 - k0) >> 6);  // 64-k steps, 4 k16-chunks each
  bf16x8 a_buf[2][4];
  const unsigned short* wp1 = (nsteps > 1) ? wp + 4 * 512 : wp;
#pragma unroll
  for (int u = 0; u < 4; ++u) {
    a_buf[0][u] = __builtin_nontemporal_load(reinterpret_cast<const bf16x8*>(wp + u * 512));
    a_buf[1][u] = __builtin_nontemporal_load(reinterpret_cast<const bf16x8*>(wp1 + u * 512));
  }
  wp += 2 * 4 * 512;

#define XRG_STEP(BUF)                                                                         \
  {                                                                                           \
    const long long kk = (long long)s * 64;                                                   \
    _Pragma("unroll")                                                                         \
    for (int u = 0; u < 4; ++u) {                                                             \
      bf16x8 bb[MT];                                                                          \
      _Pragma("unroll")                                                                       \
      for (int t = 0; t < MT; ++t)                                                            \
        bb[t] = *reinterpret_cast<const bf16x8*>(xt[t] + kk + u * 16);                        \
      _Pragma("unroll")                                                                       \
      for (int t = 0; t < MT; ++t)                                                            \
        acc[t] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(a_buf[BUF][u], bb[t], acc[t], 0, 0, 0); \
    }                                                                                         \
    if (s + 2 < nsteps) {                                                                     \
      _Pragma("unroll")                                                                       \
      for (int u = 0; u < 4; ++u)                                                             \
        a_buf[BUF][u] = __builtin_nontemporal_load(reinterpret_cast<const bf16x8*>(wp + u * 512)); \
      wp += 4 * 512;                                                                          \
    }                                                                                         \
  }

  int s = 0;
  while (s + 2 <= nsteps) {
    XRG_STEP(0);
    ++s;
    XRG_STEP(1);
    ++s;
  }
  if (s < nsteps) XRG_STEP(0);
#undef XRG_STEP

  const int m_local = lane & 31;
  const int rows_total = gridDim.y * MT * 32;
  const int nbase = tile * 128 + wv * 32 + 4 * (lane >> 5);
#pragma unroll
  for (int t = 0; t < MT; ++t) {
    const int m = e * MT * 32 + t * 32 + m_local;
    if (SPLIT) {
      float* prow = P + ((size_t)split * rows_total + m) * N;
#pragma unroll
      for (int g = 0; g < 4; ++g) {
        floatx4 v4;
#pragma unroll
        for (int j = 0; j < 4; ++j) v4[j] = acc[t][g * 4 + j];
        *reinterpret_cast<floatx4*>(prow + nbase + g * 8) = v4;
      }
    } else {
      unsigned short* yrow = Y + (size_t)m * N;
#pragma unroll
      for (int g = 0; g < 4; ++g) {
        unsigned short o[4];
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          float v = acc[t][g * 4 + j];
          if (bias) v += b2f(bias[nbase + g * 8 + j]);
          o[j] = f2b(v);
        }
        *reinterpret_cast<unsigned long long*>(yrow + nbase + g * 8) =
            *reinterpret_cast<unsigned long long*>(o);
      }
    }
  }
}

// fp8 (OCP e4m3) W8A8 variant: same structure as the bf16 packed kernel but
// operands are e4m3 with per-output-channel weight scales s_w[n] and
// per-token activation scales s_x[m] (dynamic, computed by quant_fp8_rows).
// v_mfma_f32_32x32x16_fp8_fp8 has the SAME fragment geometry as the bf16
// form (8 elements/lane), so the prepack layout carries over at half the
// bytes — decode GEMMs are weight-bandwidth-bound, so fp8 approaches 2x.
// Opt-in serving mode (XOT_FP8_GEMM=1); the benchmark path stays bf16.
// ---------------------------------------------------------------------------

typedef __attribute__((ext_vector_type(8))) char fp8x8;

DEVINL long as_i64(fp8x8 v) { return *reinterpret_cast<long*>(&v); }

template <int MT, bool SPLIT>
__global__ __launch_bounds__(256) void skinny_gemm_fp8_kernel(
    const unsigned char* __restrict__ Wp, const unsigned char* __restrict__ X8,
    const float* __restrict__ sw, const float* __restrict__ sx,
    unsigned short* __restrict__ Y, float* __restrict__ P,
    const unsigned short* __restrict__ bias,
    int N, long long K, int kc, int nsplit) {
  const int ntiles = N >> 7;
  const int tile = blockIdx.x % ntiles;
  const int split = blockIdx.x / ntiles;
  const int e = blockIdx.y;  // grouped mode (MoE): expert index
  Wp += (size_t)e * (size_t)N * (size_t)K;
  X8 += (size_t)e * (size_t)(MT * 32) * (size_t)K;
  const long long k0 = (long long)split * kc;
  const long long k1 = min(k0 + (long long)kc, K);
  if (k0 >= k1) return;
  const int lane = threadIdx.x & 63;
  const int wv = threadIdx.x >> 6;
  const int tid = threadIdx.x;

  __shared__ unsigned char xs8[MT * 32 * 72];  // fp8 rows, 72 B stride (64 + 8 pad)

  floatx16 acc[MT];
#pragma unroll
  for (int t = 0; t < MT; ++t) acc[t] = (floatx16)(0.f);

  const int n32 = tile * 4 + wv;
  const unsigned char* wp = Wp + ((size_t)n32 * (K >> 4) + (k0 >> 4)) * 512 + (size_t)lane * 8;
  // X8 staging: thread tid covers 8-byte piece q (8 of them per 64-k row)
  const int xr = tid >> 3, xq = tid & 7;
  const unsigned char* xp = X8 + (size_t)xr * K + k0 + xq * 8;
  const int xs_off = xr * 72 + xq * 8;

  const int nsteps = (int)((k1 - k0) >> 6);
  unsigned long long xv[MT];
  fp8x8 a_buf[2][4];

  const unsigned char* wp1 = (nsteps > 1) ? wp + 4 * 512 : wp;
#pragma unroll
  for (int t = 0; t < MT; ++t) xv[t] = *(const unsigned long long*)(xp + (size_t)t * 32 * K);
#pragma unroll
  for (int u = 0; u < 4; ++u) {
    a_buf[0][u] = __builtin_nontemporal_load(reinterpret_cast<const fp8x8*>(wp + u * 512));
    a_buf[1][u] = __builtin_nontemporal_load(reinterpret_cast<const fp8x8*>(wp1 + u * 512));
  }
  wp += 8 * 512;
#pragma unroll
  for (int t = 0; t < MT; ++t) *(unsigned long long*)(xs8 + t * 32 * 72 + xs_off) = xv[t];
  __syncthreads();

#define SGF_STEP(BUF)                                                                          \
  {                                                                                            \
    const bool last = (s == nsteps - 1);                                                       \
    if (!last) {                                                                               \
      _Pragma("unroll")                                                                        \
      for (int t = 0; t < MT; ++t)                                                             \
        xv[t] = *(const unsigned long long*)(xp + (size_t)t * 32 * K + (s + 1) * 64);          \
    }                                                                                          \
    _Pragma("unroll")                                                                          \
    for (int u = 0; u < 4; ++u) {                                                              \
      _Pragma("unroll")                                                                        \
      for (int t = 0; t < MT; ++t) {                                                           \
        const fp8x8 b = *reinterpret_cast<const fp8x8*>(                                       \
            xs8 + t * 32 * 72 + (lane & 31) * 72 + u * 16 + (lane >> 5) * 8);                  \
        acc[t] = __builtin_amdgcn_mfma_f32_32x32x16_fp8_fp8(                                   \
            as_i64(a_buf[BUF][u]), as_i64(b), acc[t], 0, 0, 0);                                \
      }                                                                                        \
    }                                                                                          \
    if (s + 2 < nsteps) {                                                                      \
      _Pragma("unroll")                                                                        \
      for (int u = 0; u < 4; ++u)                                                              \
        a_buf[BUF][u] = __builtin_nontemporal_load(reinterpret_cast<const fp8x8*>(wp + u * 512)); \
      wp += 4 * 512;                                                                           \
    }                                                                                          \
    if (!last) {                                                                               \
      __syncthreads();                                                                         \
      _Pragma("unroll")                                                                        \
      for (int t = 0; t < MT; ++t) *(unsigned long long*)(xs8 + t * 32 * 72 + xs_off) = xv[t]; \
      __syncthreads();                                                                         \
    }                                                                                          \
  }

  int s = 0;
  while (s + 2 <= nsteps) {
    SGF_STEP(0);
    ++s;
    SGF_STEP(1);
    ++s;
  }
  if (s < nsteps) SGF_STEP(0);
#undef SGF_STEP

  // epilogue: dequantize acc * s_x[m] * s_w[n]
  const int m_local = lane & 31;
  const int rows_total = gridDim.y * MT * 32;
  const int nbase = tile * 128 + wv * 32 + 4 * (lane >> 5);
#pragma unroll
  for (int t = 0; t < MT; ++t) {
    const int m = e * MT * 32 + t * 32 + m_local;
    const float sxm = sx[m];
    if (SPLIT) {
      float* prow = P + ((size_t)split * rows_total + m) * N;
#pragma unroll
      for (int g = 0; g < 4; ++g) {
        floatx4 v4;
#pragma unroll
        for (int j = 0; j < 4; ++j)
          v4[j] = acc[t][g * 4 + j] * sxm * sw[(size_t)e * N + nbase + g * 8 + j];
        *reinterpret_cast<floatx4*>(prow + nbase + g * 8) = v4;
      }
    } else {
      unsigned short* yrow = Y + (size_t)m * N;
#pragma unroll
      for (int g = 0; g < 4; ++g) {
        unsigned short o[4];
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          float v = acc[t][g * 4 + j] * sxm * sw[(size_t)e * N + nbase + g * 8 + j];
          if (bias) v += b2f(bias[nbase + g * 8 + j]);
          o[j] = f2b(v);
        }
        *reinterpret_cast<unsigned long long*>(yrow + nbase + g * 8) =
            *reinterpret_cast<unsigned long long*>(o);
      }
    }
  }
}

// per-row dynamic e4m3 quantization: x [M, K] bf16 -> x8 [M, K] + s_x [M]
// (s_x = rowmax/448; one 256-thread workgroup per row, K <= 64K)
__global__ __launch_bounds__(256) void quant_fp8_rows_kernel(
    const unsigned short* __restrict__ x, unsigned char* __restrict__ x8,
    float* __restrict__ sx, long long K) {
  const long long row = blockIdx.x;
  const unsigned short* xr = x + row * K;
  unsigned char* qr = x8 + row * K;
  float mx = 0.f;
  for (long long i = threadIdx.x * 8; i < K; i += 256 * 8) {
    ushort8 v = *(const ushort8*)(xr + i);
#pragma unroll
    for (int j = 0; j < 8; ++j) mx = fmaxf(mx, fabsf(b2f(v[j])));
  }
#pragma unroll
  for (int m = 32; m > 0; m >>= 1) mx = fmaxf(mx, __shfl_xor(mx, m));
  __shared__ float red[4];
  if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = mx;
  __syncthreads();
  const float scale = fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3])) / 448.f;
  const float inv = (scale > 0.f) ? 1.f / scale : 0.f;
  if (threadIdx.x == 0) sx[row] = (scale > 0.f) ? scale : 1.f;
  for (long long i = threadIdx.x * 8; i < K; i += 256 * 8) {
    ushort8 v = *(const ushort8*)(xr + i);
    unsigned char o[8];
#pragma unroll
    for (int j = 0; j < 8; j += 2) {
      const float a = b2f(v[j]) * inv, b = b2f(v[j + 1]) * inv;
      const unsigned short pk = (unsigned short)__builtin_amdgcn_cvt_pk_fp8_f32(a, b, 0, false);
      o[j] = (unsigned char)(pk & 0xff);
      o[j + 1] = (unsigned char)(pk >> 8);
    }
    *(unsigned long long*)(qr + i) = *(unsigned long long*)o;
  }
}

// combine fp32 split-K partials [S, M, N] -> bf16 [M, N] (+bias)
__global__ __launch_bounds__(256) void skinny_combine_kernel(
    const float* __restrict__ P, unsigned short* __restrict__ Y,
    const unsigned short* __restrict__ bias, long long MN, long long N, int nsplit) {
  const long long stride = (long long)gridDim.x * blockDim.x;
  for (long long i = blockIdx.x * (long long)blockDim.x + threadIdx.x; i * 4 < MN; i += stride) {
    const long long base = i * 4;
    floatx4 s = *reinterpret_cast<const floatx4*>(P + base);
    for (int sp = 1; sp < nsplit; ++sp) {
      floatx4 v = *reinterpret_cast<const floatx4*>(P + (size_t)sp * MN + base);
#pragma unroll
      for (int j = 0; j < 4; ++j) s[j] += v[j];
    }
    unsigned short o[4];
    const long long ncol = base % N;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      float v = s[j];
      if (bias) v += b2f(bias[ncol + j]);
      o[j] = f2b(v);
    }
    *reinterpret_cast<unsigned long long*>(Y + base) = *reinterpret_cast<unsigned long long*>(o);
  }
}

// ===========================================================================
// host bindings
// ===========================================================================

#define CHK(x) TORCH_CHECK(x, #x)

static inline hipStream_t cur_stream() {
  return (hipStream_t)c10::hip::getCurrentHIPStream().stream();
}

// split-K tile threshold for the skinny GEMMs: if the n-tile grid alone
// reaches ~1.5 blocks/CU (384 on MI355X's 256 CUs), splitting K only adds
// partial-write + combine overhead (measured: gate_up 448 tiles 176 -> 162 us
// unsplit); below it, split K until ~2 blocks/CU. Overridable for tuning.
static int skinny_target_blocks() {
  static int t = [] {
    const char* e = getenv("XOT_SKINNY_TARGET");
    return e ? atoi(e) : 384;
  }();
  return t;
}

torch::Tensor rmsnorm(torch::Tensor x, torch::Tensor w, double eps, double w_bias) {
  CHK(x.is_cuda() && x.dtype() == torch::kBFloat16 && x.is_contiguous());
  const int D = x.size(-1);
  CHK(D % 8 == 0 && D <= 16384);
  const int rows = x.numel() / D;
  auto out = torch::empty_like(x);
  hipLaunchKernelGGL((rmsnorm_kernel<false>), dim3(rows), dim3(256), 0, cur_stream(),
                     (const unsigned short*)x.data_ptr(), nullptr,
                     (const unsigned short*)w.data_ptr(), (unsigned short*)out.data_ptr(),
                     nullptr, D, (float)eps, (float)w_bias);
  return out;
}

std::vector<torch::Tensor> rmsnorm_residual(torch::Tensor x, torch::Tensor res, torch::Tensor w, double eps,
                                            double w_bias) {
  CHK(x.is_cuda() && x.dtype() == torch::kBFloat16 && x.is_contiguous() && res.is_contiguous());
  const int D = x.size(-1);
  CHK(D % 8 == 0 && D <= 16384);
  const int rows = x.numel() / D;
  auto out = torch::empty_like(x);
  auto res_out = torch::empty_like(x);
  hipLaunchKernelGGL((rmsnorm_kernel<true>), dim3(rows), dim3(256), 0, cur_stream(),
                     (const unsigned short*)x.data_ptr(), (const unsigned short*)res.data_ptr(),
                     (const unsigned short*)w.data_ptr(), (unsigned short*)out.data_ptr(),
                     (unsigned short*)res_out.data_ptr(), D, (float)eps, (float)w_bias);
  return {out, res_out};
}

void rope_qkv_append(torch::Tensor qkv, torch::Tensor cos, torch::Tensor sin,
                     torch::Tensor positions, torch::Tensor kc, torch::Tensor vc,
                     int64_t n_heads, int64_t n_kv_heads, int64_t head_dim,
                     c10::optional<torch::Tensor> kp, c10::optional<torch::Tensor> vp,
                     c10::optional<torch::Tensor> q_norm, c10::optional<torch::Tensor> k_norm,
                     double norm_eps,
                     c10::optional<torch::Tensor> k_scale, c10::optional<torch::Tensor> v_scale) {
  CHK(qkv.is_cuda() && qkv.dtype() == torch::kBFloat16 && qkv.is_contiguous());
  CHK(kc.is_contiguous() && vc.is_contiguous());
  CHK(positions.dtype() == torch::kInt32 && positions.is_cuda());
  const int B = qkv.size(0), S = qkv.size(1);
  const int H = (int)n_heads, KVH = (int)n_kv_heads, hd = (int)head_dim;
  const int T = kc.size(2);
  CHK(qkv.size(2) == (H + 2 * KVH) * hd);
  CHK(hd <= 128 && hd % 2 == 0);
  const int npos = (int)positions.numel();
  CHK(npos == S || npos == B * S);
  CHK(positions.is_contiguous());
  unsigned short* kpc = nullptr;
  unsigned short* vpc = nullptr;
  unsigned char* kp8 = nullptr;
  unsigned char* vp8 = nullptr;
  float* skp = nullptr;
  float* svp = nullptr;
  int T32 = 0;
  if (kp.has_value() && vp.has_value()) {
    CHK(hd == 128 && kp->is_contiguous() && vp->is_contiguous());
    T32 = (int)kp->size(2) * 16;
    if (kp->dtype() == torch::kUInt8) {
      // fp8 packed mode: per-row e4m3 scales required
      CHK(k_scale.has_value() && v_scale.has_value());
      CHK(k_scale->dtype() == torch::kFloat32 && k_scale->is_contiguous());
      CHK(v_scale->dtype() == torch::kFloat32 && v_scale->is_contiguous());
      kp8 = (unsigned char*)kp->data_ptr();
      vp8 = (unsigned char*)vp->data_ptr();
      skp = k_scale->data_ptr<float>();
      svp = v_scale->data_ptr<float>();
    } else {
      kpc = (unsigned short*)kp->data_ptr();
      vpc = (unsigned short*)vp->data_ptr();
    }
  }
  const unsigned short* qnp = nullptr;
  const unsigned short* knp = nullptr;
  if (q_norm.has_value()) {
    CHK(q_norm->is_contiguous() && q_norm->dtype() == torch::kBFloat16 && q_norm->numel() == hd);
    qnp = (const unsigned short*)q_norm->data_ptr();
  }
  if (k_norm.has_value()) {
    CHK(k_norm->is_contiguous() && k_norm->dtype() == torch::kBFloat16 && k_norm->numel() == hd);
    knp = (const unsigned short*)k_norm->data_ptr();
  }
  const int waves = B * S * (H + 2 * KVH);
  const int blocks = (waves + 3) / 4;
  hipLaunchKernelGGL(rope_qkv_append_kernel, dim3(blocks), dim3(256), 0, cur_stream(),
                     (unsigned short*)qkv.data_ptr(), cos.data_ptr<float>(), sin.data_ptr<float>(),
                     positions.data_ptr<int>(), (unsigned short*)kc.data_ptr(),
                     (unsigned short*)vc.data_ptr(), B, S, H, KVH, hd, T, kpc, vpc, T32,
                     qnp, knp, (float)norm_eps, npos, kp8, vp8, skp, svp);
}

template <int HD>
static void launch_attn_partial(int NQ, const unsigned short* q, const unsigned short* kc,
                                const unsigned short* vc, const int* sl, float* ws_o, float* ws_ml,
                                int B, int H, int KVH, int T, int nsplit, int qh0, float scale,
                                long long q_stride, hipStream_t stream) {
  const dim3 grid(B * KVH * nsplit), block(256);
#define CASE(NQV) \
  case NQV: \
    hipLaunchKernelGGL((attn_decode_partial<NQV, HD>), grid, block, 0, stream, q, kc, vc, sl, \
                       ws_o, ws_ml, B, H, KVH, T, nsplit, qh0, scale, q_stride); \
    break;
  switch (NQ) {
    CASE(1) CASE(2) CASE(3) CASE(4) CASE(5) CASE(6) CASE(7) CASE(8)
    default: TORCH_CHECK(false, "unsupported q-heads-per-kv-head slice: ", NQ);
  }
#undef CASE
}

torch::Tensor attn_decode(torch::Tensor q, torch::Tensor kc, torch::Tensor vc, torch::Tensor seq_lens) {
  // q may be a strided view into the packed qkv tensor: [B, 1, H, hd] with an
  // arbitrary batch stride but contiguous (head, dim) rows.
  CHK(q.is_cuda() && q.dtype() == torch::kBFloat16);
  CHK(q.stride(3) == 1 && q.stride(2) == q.size(3));
  CHK(seq_lens.dtype() == torch::kInt32 && seq_lens.is_cuda());
  const int B = q.size(0), H = q.size(2), hd = q.size(3);
  const long long q_stride = q.stride(0);
  const int KVH = kc.size(1), T = kc.size(2);
  TORCH_CHECK(hd == 64 || hd == 128, "attn_decode: head_dim must be 64 or 128, got ", hd);
  const int rep = H / KVH;
  // fill the 256 CUs: at least ~512 workgroups, chunks >= 128 positions
  int nsplit = std::max(1, 512 / std::max(1, B * KVH));
  nsplit = std::min<int>(nsplit, std::max(1, (T + 127) / 128));
  auto opts = torch::TensorOptions().dtype(torch::kFloat32).device(q.device());
  auto ws_o = torch::empty({(long)B * H * nsplit * hd}, opts);
  auto ws_ml = torch::empty({(long)B * H * nsplit * 2}, opts);
  auto out = torch::empty({q.size(0), q.size(1), q.size(2), q.size(3)},
                          torch::TensorOptions().dtype(torch::kBFloat16).device(q.device()));
  const float scale = 1.0f / sqrtf((float)hd);
  auto stream = cur_stream();
  for (int qh0 = 0; qh0 < rep; qh0 += 8) {
    const int nq = std::min(8, rep - qh0);
    if (hd == 128)
      launch_attn_partial<128>(nq, (const unsigned short*)q.data_ptr(), (const unsigned short*)kc.data_ptr(),
                               (const unsigned short*)vc.data_ptr(), seq_lens.data_ptr<int>(),
                               ws_o.data_ptr<float>(), ws_ml.data_ptr<float>(), B, H, KVH, T, nsplit, qh0,
                               scale, q_stride, stream);
    else
      launch_attn_partial<64>(nq, (const unsigned short*)q.data_ptr(), (const unsigned short*)kc.data_ptr(),
                              (const unsigned short*)vc.data_ptr(), seq_lens.data_ptr<int>(),
                              ws_o.data_ptr<float>(), ws_ml.data_ptr<float>(), B, H, KVH, T, nsplit, qh0,
                              scale, q_stride, stream);
  }
  if (hd == 128)
    hipLaunchKernelGGL((attn_decode_merge<128>), dim3(B * H), dim3(128), 0, stream,
                       ws_o.data_ptr<float>(), ws_ml.data_ptr<float>(), (unsigned short*)out.data_ptr(), nsplit);
  else
    hipLaunchKernelGGL((attn_decode_merge<64>), dim3(B * H), dim3(128), 0, stream,
                       ws_o.data_ptr<float>(), ws_ml.data_ptr<float>(), (unsigned short*)out.data_ptr(), nsplit);
  return out;
}

// q: [B, 1, H, 128] (strided batch OK); kp/vp: the packed cache copies.
torch::Tensor attn_decode_mfma(torch::Tensor q, torch::Tensor kp, torch::Tensor vp,
                               torch::Tensor seq_lens, int64_t t_capacity,
                               double scale_in, double softcap, int64_t window,
                               c10::optional<torch::Tensor> k_scale,
                               c10::optional<torch::Tensor> v_scale) {
  CHK(q.is_cuda() && q.dtype() == torch::kBFloat16);
  CHK(q.stride(3) == 1 && q.stride(2) == q.size(3));
  CHK(seq_lens.dtype() == torch::kInt32 && seq_lens.is_cuda());
  CHK(kp.is_contiguous() && vp.is_contiguous());
  const bool fp8 = kp.dtype() == torch::kUInt8;
  const float* skp = nullptr;
  const float* svp = nullptr;
  if (fp8) {
    CHK(k_scale.has_value() && v_scale.has_value());
    skp = k_scale->data_ptr<float>();
    svp = v_scale->data_ptr<float>();
  }
  const int B = q.size(0), H = q.size(2), hd = q.size(3);
  TORCH_CHECK(hd == 128, "attn_decode_mfma requires head_dim 128");
  const int KVH = kp.size(1);
  const int T32 = kp.size(2) * 16;
  const long long q_stride = q.stride(0);
  // one wave per (b, kvh, split); target >= ~2048 waves so 16 waves/CU keep
  // the packed-cache stream deep while chunks stay >= 32 positions
  int nsplit = 1;
  while (B * KVH * nsplit * 2 < 4096 && (T32 / (nsplit * 2)) >= 32 && nsplit < 32) nsplit *= 2;
  auto opts = torch::TensorOptions().dtype(torch::kFloat32).device(q.device());
  auto ws_o = torch::empty({(long)B * H * nsplit * hd}, opts);
  auto ws_ml = torch::empty({(long)B * H * nsplit * 2}, opts);
  auto out = torch::empty({q.size(0), q.size(1), q.size(2), q.size(3)},
                          torch::TensorOptions().dtype(torch::kBFloat16).device(q.device()));
  const float scale = (scale_in > 0.0) ? (float)scale_in : 1.0f / sqrtf((float)hd);
  auto stream = cur_stream();
  const int waves = B * KVH * nsplit;
  // default ON: measured -1.1 ms/step on 70B B=128 and -0.8 on 8B B=256
  const char* pf_env = getenv("XOT_ATTN_PREFETCH");
  const bool prefetch = (pf_env == nullptr) || (pf_env[0] != '0');
#define ADM_LAUNCH(PF, F8)   hipLaunchKernelGGL((attn_decode_mfma_kernel<PF, F8>), dim3((waves + 3) / 4), dim3(256), 0, stream,                      (const unsigned short*)q.data_ptr(), (const unsigned short*)kp.data_ptr(),                      (const unsigned short*)vp.data_ptr(), seq_lens.data_ptr<int>(),                      ws_o.data_ptr<float>(), ws_ml.data_ptr<float>(), B, H, KVH, T32, nsplit,                      scale, q_stride, (float)softcap, (int)window, skp, svp)
  if (prefetch && fp8) ADM_LAUNCH(true, true);
  else if (prefetch) ADM_LAUNCH(true, false);
  else if (fp8) ADM_LAUNCH(false, true);
  else ADM_LAUNCH(false, false);
#undef ADM_LAUNCH
  hipLaunchKernelGGL((attn_decode_merge<128>), dim3(B * H), dim3(128), 0, stream,
                     ws_o.data_ptr<float>(), ws_ml.data_ptr<float>(),
                     (unsigned short*)out.data_ptr(), nsplit);
  return out;
}

// q: [B, S, H, 128] (strided over b/s OK, head rows contiguous); kp/vp: the
// packed cache copies already holding positions [0, start_pos + S).
torch::Tensor attn_prefill_mfma(torch::Tensor q, torch::Tensor kp, torch::Tensor vp,
                                int64_t start_pos, double scale_in, double softcap,
                                int64_t window) {
  CHK(q.is_cuda() && q.dtype() == torch::kBFloat16);
  CHK(q.stride(3) == 1 && q.stride(2) == q.size(3));
  CHK(kp.is_contiguous() && vp.is_contiguous());
  const int B = q.size(0), S = q.size(1), H = q.size(2), hd = q.size(3);
  TORCH_CHECK(hd == 128, "attn_prefill_mfma requires head_dim 128");
  const int KVH = kp.size(1);
  const int T32 = kp.size(2) * 16;
  CHK(start_pos + S <= T32);
  auto out = torch::empty({B, S, H, hd},
                          torch::TensorOptions().dtype(torch::kBFloat16).device(q.device()));
  const float scale = (scale_in > 0.0) ? (float)scale_in : 1.0f / sqrtf((float)hd);
  const int qblocks = (S + 127) / 128;
  hipLaunchKernelGGL(attn_prefill_mfma_kernel, dim3(B * qblocks * H), dim3(256), 0, cur_stream(),
                     (const unsigned short*)q.data_ptr(), (const unsigned short*)kp.data_ptr(),
                     (const unsigned short*)vp.data_ptr(), (unsigned short*)out.data_ptr(),
                     B, S, H, KVH, T32, (int)start_pos, q.stride(0), q.stride(1), scale,
                     (float)softcap, (int)window);
  return out;
}

// logits: [T, E] fp32 gate output -> (idx int32 [T,k], w fp32 [T,k]).
std::vector<torch::Tensor> moe_route(torch::Tensor logits, c10::optional<torch::Tensor> bias,
                                     int64_t k, int64_t mode, int64_t n_group,
                                     int64_t topk_group, double routed_scale, bool norm_topk) {
  CHK(logits.is_cuda() && logits.dtype() == torch::kFloat32 && logits.is_contiguous() && logits.dim() == 2);
  const int T = logits.size(0), E = logits.size(1);
  CHK(E <= 256 && k >= 1 && k <= 8 && n_group >= 1 && n_group <= 8);
  const float* bptr = nullptr;
  if (bias.has_value()) {
    CHK(bias->is_contiguous() && bias->dtype() == torch::kFloat32 && bias->numel() == E);
    bptr = bias->data_ptr<float>();
  }
  auto iopts = torch::TensorOptions().dtype(torch::kInt32).device(logits.device());
  auto fopts = torch::TensorOptions().dtype(torch::kFloat32).device(logits.device());
  auto idx = torch::empty({(long)T, (long)k}, iopts);
  auto w = torch::empty({(long)T, (long)k}, fopts);
  hipLaunchKernelGGL(moe_route_kernel, dim3((T + 3) / 4), dim3(256), 0, cur_stream(),
                     logits.data_ptr<float>(), bptr, idx.data_ptr<int>(), w.data_ptr<float>(),
                     T, E, (int)k, (int)mode, (int)n_group, (int)topk_group,
                     (float)routed_scale, norm_topk ? 1 : 0);
  return {idx, w};
}

// idx: [T, k] int32 expert choices -> (gather_tok int32 [E*C], inv_pos
// int32 [T, k]). One workgroup (counting sort in LDS).
std::vector<torch::Tensor> moe_build(torch::Tensor idx, int64_t E, int64_t C) {
  CHK(idx.is_cuda() && idx.dtype() == torch::kInt32 && idx.is_contiguous() && idx.dim() == 2);
  const int T = idx.size(0), k = idx.size(1);
  CHK(E <= 256 && T * k <= 8192 && T <= C);
  auto opts = torch::TensorOptions().dtype(torch::kInt32).device(idx.device());
  auto gather_tok = torch::empty({E * C}, opts);
  auto inv_pos = torch::empty({T, k}, opts);
  hipLaunchKernelGGL(moe_build_kernel, dim3(1), dim3(256), 0, cur_stream(),
                     idx.data_ptr<int>(), gather_tok.data_ptr<int>(),
                     inv_pos.data_ptr<int>(), T, k, (int)E, (int)C);
  return {gather_tok, inv_pos};
}

// y: [E*C, D] bf16 expert outputs, inv_pos [T,k] int32, w [T,k] fp32 ->
// out [T, D] bf16 (deterministic weighted combine, no atomics).
torch::Tensor moe_combine(torch::Tensor y, torch::Tensor inv_pos, torch::Tensor w) {
  CHK(y.is_cuda() && y.dtype() == torch::kBFloat16 && y.is_contiguous());
  CHK(inv_pos.dtype() == torch::kInt32 && inv_pos.is_contiguous());
  CHK(w.dtype() == torch::kFloat32 && w.is_contiguous());
  const int T = inv_pos.size(0), k = inv_pos.size(1);
  const int D = y.size(-1);
  CHK(D % 8 == 0);
  auto out = torch::empty({(long)T, (long)D},
                          torch::TensorOptions().dtype(torch::kBFloat16).device(y.device()));
  const long long n8 = (long long)T * (D / 8);
  const int blocks = (int)std::min<long long>(1024, (n8 + 255) / 256);
  hipLaunchKernelGGL(moe_combine_kernel, dim3(blocks), dim3(256), 0, cur_stream(),
                     (const unsigned short*)y.data_ptr(), inv_pos.data_ptr<int>(),
                     w.data_ptr<float>(), (unsigned short*)out.data_ptr(), T, k, D);
  return out;
}

// q: [B, 1, H, nope+64] bf16 contiguous (raw projections, nope part is the
// un-roped passthrough); q_lat: [B, 1, H, 512] absorbed latent query;
// returns qfull [B, H, 576] with the roped 64-dim tail appended.
std::vector<torch::Tensor> mla_q_prep(torch::Tensor q, torch::Tensor q_lat, torch::Tensor cos,
                                      torch::Tensor sin, torch::Tensor positions,
                                      int64_t nope, bool interleave, bool fp8) {
  CHK(q.is_cuda() && q.dtype() == torch::kBFloat16 && q.is_contiguous());
  CHK(q_lat.is_cuda() && q_lat.dtype() == torch::kBFloat16 && q_lat.is_contiguous());
  CHK(positions.dtype() == torch::kInt32 && positions.is_contiguous());
  const int B = q.size(0), H = q.size(2);
  CHK(q.size(1) == 1 && q.size(3) == nope + MLA_ROPE);
  CHK(q_lat.numel() == (long long)B * H * MLA_LAT);
  const int npos = (int)positions.numel();
  CHK(npos == 1 || npos == B);
  const int waves = B * H;
  if (fp8) {
    auto q8 = torch::empty({(long)B, (long)H, (long)MLA_DQK},
                           torch::TensorOptions().dtype(torch::kUInt8).device(q.device()));
    auto sq = torch::empty({(long)B, (long)H},
                           torch::TensorOptions().dtype(torch::kFloat32).device(q.device()));
    hipLaunchKernelGGL(mla_q_prep_kernel, dim3((waves + 3) / 4), dim3(256), 0, cur_stream(),
                       (const unsigned short*)q.data_ptr(), (const unsigned short*)q_lat.data_ptr(),
                       cos.data_ptr<float>(), sin.data_ptr<float>(), positions.data_ptr<int>(),
                       nullptr, B, H, (long long)H * (nope + MLA_ROPE),
                       (int)nope, interleave ? 1 : 0, npos,
                       (unsigned char*)q8.data_ptr(), sq.data_ptr<float>());
    return {q8, sq};
  }
  auto qfull = torch::empty({(long)B, (long)H, (long)MLA_DQK},
                            torch::TensorOptions().dtype(torch::kBFloat16).device(q.device()));
  hipLaunchKernelGGL(mla_q_prep_kernel, dim3((waves + 3) / 4), dim3(256), 0, cur_stream(),
                     (const unsigned short*)q.data_ptr(), (const unsigned short*)q_lat.data_ptr(),
                     cos.data_ptr<float>(), sin.data_ptr<float>(), positions.data_ptr<int>(),
                     (unsigned short*)qfull.data_ptr(), B, H, (long long)H * (nope + MLA_ROPE),
                     (int)nope, interleave ? 1 : 0, npos, nullptr, nullptr);
  return {qfull};
}

// ckv: [B, S, 576] raw kv_a output; w: [512] bf16 norm weight; cos/sin
// fp32 [maxT, 32]; lat_c/rot_c: the plain caches viewed [B, T, 512]/[B, T, 64].
void mla_prep_append(torch::Tensor ckv, torch::Tensor w, torch::Tensor cos,
                     torch::Tensor sin, torch::Tensor positions,
                     torch::Tensor lat_c, torch::Tensor rot_c,
                     torch::Tensor kp, torch::Tensor vp, double eps, bool interleave,
                     c10::optional<torch::Tensor> k_scale) {
  CHK(ckv.is_cuda() && ckv.dtype() == torch::kBFloat16 && ckv.is_contiguous());
  CHK(w.dtype() == torch::kBFloat16 && w.is_contiguous() && w.numel() == MLA_LAT);
  CHK(positions.dtype() == torch::kInt32 && positions.is_contiguous());
  CHK(lat_c.is_contiguous() && rot_c.is_contiguous() && kp.is_contiguous() && vp.is_contiguous());
  const int B = ckv.size(0), S = ckv.size(1);
  CHK(ckv.size(2) == MLA_DQK);
  const int T = lat_c.numel() / (B * MLA_LAT);
  const int T32 = (int)kp.size(1) * 16;
  const int npos = (int)positions.numel();
  CHK(npos == S || npos == B * S);
  const int waves = B * S;
  unsigned short* kpc = nullptr;
  unsigned short* vpc = nullptr;
  unsigned char* kp8 = nullptr;
  unsigned char* vp8 = nullptr;
  float* ksp = nullptr;
  if (kp.dtype() == torch::kUInt8) {
    CHK(k_scale.has_value() && k_scale->dtype() == torch::kFloat32 && k_scale->is_contiguous());
    kp8 = (unsigned char*)kp.data_ptr();
    vp8 = (unsigned char*)vp.data_ptr();
    ksp = k_scale->data_ptr<float>();
  } else {
    kpc = (unsigned short*)kp.data_ptr();
    vpc = (unsigned short*)vp.data_ptr();
  }
  hipLaunchKernelGGL(mla_prep_append_kernel, dim3((waves + 3) / 4), dim3(256), 0, cur_stream(),
                     (const unsigned short*)ckv.data_ptr(), (const unsigned short*)w.data_ptr(),
                     cos.data_ptr<float>(), sin.data_ptr<float>(), positions.data_ptr<int>(),
                     (unsigned short*)lat_c.data_ptr(), (unsigned short*)rot_c.data_ptr(),
                     kpc, vpc, B, S, T, T32, (float)eps, interleave ? 1 : 0, npos,
                     kp8, vp8, ksp);
}

// lat: [B, S, 512] bf16 (post-RMSNorm latent), rot: [B, S, 64] bf16 (roped
// shared key); kp: [B, T32/16, 18, 64, 8], vp: [B, 32, T32/32, 64, 8].
void mla_append(torch::Tensor lat, torch::Tensor rot, torch::Tensor positions,
                torch::Tensor kp, torch::Tensor vp) {
  CHK(lat.is_cuda() && lat.dtype() == torch::kBFloat16 && lat.is_contiguous());
  CHK(rot.is_cuda() && rot.dtype() == torch::kBFloat16 && rot.is_contiguous());
  CHK(positions.dtype() == torch::kInt32 && positions.is_cuda() && positions.is_contiguous());
  CHK(kp.is_contiguous() && vp.is_contiguous());
  const int B = lat.size(0), S = lat.size(1);
  CHK(lat.size(2) == MLA_LAT && rot.size(2) == MLA_ROPE);
  const int T32 = (int)kp.size(1) * 16;
  const int npos = (int)positions.numel();
  CHK(npos == S || npos == B * S);
  const int waves = B * S;
  hipLaunchKernelGGL(mla_append_kernel, dim3((waves + 3) / 4), dim3(256), 0, cur_stream(),
                     (const unsigned short*)lat.data_ptr(), (const unsigned short*)rot.data_ptr(),
                     positions.data_ptr<int>(), (unsigned short*)kp.data_ptr(),
                     (unsigned short*)vp.data_ptr(), B, S, T32, npos);
}

// q: [B, H, 576] bf16 (absorbed latent+rope query); returns out_lat
// [B, H, 512] bf16 (latent-space attention output, pre kv_b-v expansion).
torch::Tensor attn_decode_mla(torch::Tensor q, torch::Tensor kp, torch::Tensor vp,
                              torch::Tensor seq_lens, double scale_in,
                              c10::optional<torch::Tensor> q_scale,
                              c10::optional<torch::Tensor> k_scale) {
  const bool fp8 = kp.dtype() == torch::kUInt8;
  CHK(q.is_cuda() && q.is_contiguous());
  CHK(fp8 ? (q.dtype() == torch::kUInt8) : (q.dtype() == torch::kBFloat16));
  CHK(seq_lens.dtype() == torch::kInt32 && seq_lens.is_cuda());
  CHK(kp.is_contiguous() && vp.is_contiguous());
  const int B = q.size(0), H = q.size(1);
  CHK(q.size(2) == MLA_DQK);
  const int T32 = (int)kp.size(1) * 16;
  const int hgroups = (H + 15) / 16;
  // fill the chip: B*hgroups is small for lite MLA configs (64 x 1), so
  // split the kv range aggressively — one 32-pos tile per split is fine
  // (empty splits merge as -inf partials). 128 WGs on 256 CUs measured
  // 1.1 TB/s; 256+ WGs is the floor for the packed stream.
  int nsplit = 1;
  while (B * hgroups * nsplit * 2 < 4096 && (T32 / (nsplit * 2)) >= 16 && nsplit < 64) nsplit *= 2;
  auto opts = torch::TensorOptions().dtype(torch::kFloat32).device(q.device());
  auto ws_o = torch::empty({(long)B * H * nsplit * MLA_LAT}, opts);
  auto ws_ml = torch::empty({(long)B * H * nsplit * 2}, opts);
  auto out = torch::empty({(long)B, (long)H, (long)MLA_LAT},
                          torch::TensorOptions().dtype(torch::kBFloat16).device(q.device()));
  const float scale = (scale_in > 0.0) ? (float)scale_in : 1.0f / sqrtf((float)MLA_DQK);
  auto stream = cur_stream();
  const int waves = B * hgroups * nsplit;
  const float* sqp = nullptr;
  const float* ksp = nullptr;
  if (fp8) {
    CHK(q_scale.has_value() && k_scale.has_value());
    sqp = q_scale->data_ptr<float>();
    ksp = k_scale->data_ptr<float>();
  }
  if (fp8)
    hipLaunchKernelGGL((attn_decode_mla_kernel<true>), dim3((waves + 3) / 4), dim3(256), 0, stream,
                       (const unsigned short*)q.data_ptr(), (const unsigned short*)kp.data_ptr(),
                       (const unsigned short*)vp.data_ptr(), seq_lens.data_ptr<int>(),
                       ws_o.data_ptr<float>(), ws_ml.data_ptr<float>(), B, H, T32, nsplit, scale,
                       sqp, ksp);
  else
    hipLaunchKernelGGL((attn_decode_mla_kernel<false>), dim3((waves + 3) / 4), dim3(256), 0, stream,
                       (const unsigned short*)q.data_ptr(), (const unsigned short*)kp.data_ptr(),
                       (const unsigned short*)vp.data_ptr(), seq_lens.data_ptr<int>(),
                       ws_o.data_ptr<float>(), ws_ml.data_ptr<float>(), B, H, T32, nsplit, scale);
  hipLaunchKernelGGL(attn_decode_merge512, dim3(B * H), dim3(256), 0, stream,
                     ws_o.data_ptr<float>(), ws_ml.data_ptr<float>(),
                     (unsigned short*)out.data_ptr(), nsplit);
  return out;
}

torch::Tensor mfma16_probe(torch::Tensor a, torch::Tensor b) {
  CHK(a.is_cuda() && a.dtype() == torch::kBFloat16 && a.is_contiguous() && a.numel() == 16 * 32);
  CHK(b.is_cuda() && b.dtype() == torch::kBFloat16 && b.is_contiguous() && b.numel() == 32 * 16);
  auto d = torch::empty({16, 16}, torch::TensorOptions().dtype(torch::kFloat32).device(a.device()));
  hipLaunchKernelGGL(mfma16_probe_kernel, dim3(1), dim3(64), 0, cur_stream(),
                     (const unsigned short*)a.data_ptr(), (const unsigned short*)b.data_ptr(),
                     d.data_ptr<float>());
  return d;
}

torch::Tensor swiglu(torch::Tensor g, torch::Tensor u) {
  CHK(g.is_cuda() && g.dtype() == torch::kBFloat16 && g.is_contiguous() && u.is_contiguous());
  CHK(g.numel() % 8 == 0);
  auto out = torch::empty_like(g);
  const long long n8 = g.numel() / 8;
  const int blocks = (int)std::min<long long>(2048, (n8 + 255) / 256);
  hipLaunchKernelGGL(swiglu_kernel, dim3(blocks), dim3(256), 0, cur_stream(),
                     (const unsigned short*)g.data_ptr(), (const unsigned short*)u.data_ptr(),
                     (unsigned short*)out.data_ptr(), n8);
  return out;
}

torch::Tensor swiglu_packed(torch::Tensor gu) {
  CHK(gu.is_cuda() && gu.dtype() == torch::kBFloat16 && gu.is_contiguous());
  const int twoI = gu.size(-1);
  CHK(twoI % 16 == 0);
  const int I = twoI / 2;
  const long long rows = gu.numel() / twoI;
  auto sizes = gu.sizes().vec();
  sizes.back() = I;
  auto out = torch::empty(sizes, gu.options());
  const long long n8 = rows * (I / 8);
  const int blocks = (int)std::min<long long>(2048, (n8 + 255) / 256);
  hipLaunchKernelGGL(swiglu_packed_kernel, dim3(blocks), dim3(256), 0, cur_stream(),
                     (const unsigned short*)gu.data_ptr(), (unsigned short*)out.data_ptr(), rows, I);
  return out;
}

torch::Tensor geglu_packed(torch::Tensor gu) {
  CHK(gu.is_cuda() && gu.dtype() == torch::kBFloat16 && gu.is_contiguous());
  const int twoI = gu.size(-1);
  CHK(twoI % 16 == 0);
  const int I = twoI / 2;
  const long long rows = gu.numel() / twoI;
  auto sizes = gu.sizes().vec();
  sizes.back() = I;
  auto out = torch::empty(sizes, gu.options());
  const long long n8 = rows * (I / 8);
  const int blocks = (int)std::min<long long>(2048, (n8 + 255) / 256);
  hipLaunchKernelGGL(geglu_packed_kernel, dim3(blocks), dim3(256), 0, cur_stream(),
                     (const unsigned short*)gu.data_ptr(), (unsigned short*)out.data_ptr(), rows, I);
  return out;
}

// Y = x @ W^T (+bias). x: [M, K] bf16 contiguous rows (M <= 256, M % 32 == 0),
// w: [N, K] bf16 contiguous, bias: optional [N] bf16.
torch::Tensor skinny_gemm(torch::Tensor x, torch::Tensor w,
                          c10::optional<torch::Tensor> bias) {
  CHK(x.is_cuda() && x.dtype() == torch::kBFloat16);
  CHK(w.is_cuda() && w.dtype() == torch::kBFloat16 && w.is_contiguous());
  const long long K = w.size(1);
  const int N = (int)w.size(0);
  const long long M = x.numel() / K;
  CHK(x.is_contiguous());
  CHK(M >= 32 && M <= 256 && M % 32 == 0);
  CHK(N % 128 == 0 && K % 16 == 0);
  const unsigned short* bptr = nullptr;
  if (bias.has_value()) {
    CHK(bias->is_contiguous() && bias->dtype() == torch::kBFloat16 && bias->numel() == N);
    bptr = (const unsigned short*)bias->data_ptr();
  }
  auto sizes = x.sizes().vec();
  sizes.back() = N;
  auto y = torch::empty(sizes, x.options());
  const int ntiles = N / 128;
  // oversubscribe the 256 CUs (>=2 blocks/CU) while keeping K/SPLITK >= ~1024
  int nsplit = 1;
  while (ntiles * nsplit < skinny_target_blocks() && (K / (nsplit * 2)) >= 1024 && nsplit < 16) nsplit *= 2;
  int kc = (int)((K / nsplit + 15) / 16 * 16);
  while ((long long)kc * (nsplit - 1) >= K) nsplit--;  // drop empty splits
  auto stream = cur_stream();
  const int MT = (int)(M / 32);
  const dim3 grid(ntiles * nsplit), block(256);
#define SG_CASE(MTV) \
  case MTV: \
    if (nsplit == 1) { \
      hipLaunchKernelGGL((skinny_gemm_kernel<MTV, false>), grid, block, 0, stream, \
                         (const unsigned short*)w.data_ptr(), (const unsigned short*)x.data_ptr(), \
                         (unsigned short*)y.data_ptr(), nullptr, bptr, N, K, kc, nsplit); \
    } else { \
      hipLaunchKernelGGL((skinny_gemm_kernel<MTV, true>), grid, block, 0, stream, \
                         (const unsigned short*)w.data_ptr(), (const unsigned short*)x.data_ptr(), \
                         nullptr, P.data_ptr<float>(), nullptr, N, K, kc, nsplit); \
    } \
    break;
  if (nsplit == 1) {
    torch::Tensor P;  // unused
    switch (MT) { SG_CASE(1) SG_CASE(2) SG_CASE(3) SG_CASE(4) SG_CASE(5) SG_CASE(6) SG_CASE(7) SG_CASE(8) }
  } else {
    auto P = torch::empty({nsplit, M, (long long)N},
                          torch::TensorOptions().dtype(torch::kFloat32).device(x.device()));
    switch (MT) { SG_CASE(1) SG_CASE(2) SG_CASE(3) SG_CASE(4) SG_CASE(5) SG_CASE(6) SG_CASE(7) SG_CASE(8) }
    const long long MN = M * (long long)N;
    const int blocks = (int)std::min<long long>(2048, (MN / 4 + 255) / 256);
    hipLaunchKernelGGL(skinny_combine_kernel, dim3(blocks), dim3(256), 0, stream,
                       P.data_ptr<float>(), (unsigned short*)y.data_ptr(), bptr, MN, N, nsplit);
  }
#undef SG_CASE
  return y;
}

// Packed variant. wp: the [N/32, K/16, 64, 8] prepack of w (see
// ops.pack_decode_weight), x: [M, K] bf16, M % 32 == 0, K % 64 == 0.
torch::Tensor skinny_gemm_packed(torch::Tensor x, torch::Tensor wp, int64_t N,
                                 c10::optional<torch::Tensor> bias) {
  CHK(x.is_cuda() && x.dtype() == torch::kBFloat16 && x.is_contiguous());
  CHK(wp.is_cuda() && wp.dtype() == torch::kBFloat16 && wp.is_contiguous());
  const long long K = wp.numel() / N;
  const long long M = x.numel() / K;
  CHK(M >= 32 && M <= 256 && M % 32 == 0);
  CHK(N % 128 == 0 && K % 64 == 0);
  const unsigned short* bptr = nullptr;
  if (bias.has_value()) {
    CHK(bias->is_contiguous() && bias->dtype() == torch::kBFloat16 && bias->numel() == N);
    bptr = (const unsigned short*)bias->data_ptr();
  }
  auto sizes = x.sizes().vec();
  sizes.back() = (long)N;
  auto y = torch::empty(sizes, x.options());
  const int ntiles = (int)(N / 128);
  int nsplit = 1;
  while (ntiles * nsplit < skinny_target_blocks() && (K / (nsplit * 2)) >= 1024 && nsplit < 16) nsplit *= 2;
  int kc = (int)((K / nsplit + 63) / 64 * 64);
  while ((long long)kc * (nsplit - 1) >= K) nsplit--;
  auto stream = cur_stream();
  const int MT = (int)(M / 32);
  // BK=128 halves the staging-barrier count per byte; needs 128-aligned splits
  const bool bk128 = (K % 128 == 0) && (kc % 128 == 0) && kc >= 2048
                     && getenv("XOT_SKINNY_BK64") == nullptr;
  const dim3 grid(ntiles * nsplit), block(256);
#define SGP_CASE(MTV) \
  case MTV: \
    if (nsplit == 1) { \
      if (bk128) \
        hipLaunchKernelGGL((skinny_gemm_packed_kernel<MTV, false, 128>), grid, block, 0, stream, \
                           (const unsigned short*)wp.data_ptr(), (const unsigned short*)x.data_ptr(), \
                           (unsigned short*)y.data_ptr(), nullptr, bptr, (int)N, K, kc, nsplit); \
      else \
        hipLaunchKernelGGL((skinny_gemm_packed_kernel<MTV, false, 64>), grid, block, 0, stream, \
                           (const unsigned short*)wp.data_ptr(), (const unsigned short*)x.data_ptr(), \
                           (unsigned short*)y.data_ptr(), nullptr, bptr, (int)N, K, kc, nsplit); \
    } else { \
      if (bk128) \
        hipLaunchKernelGGL((skinny_gemm_packed_kernel<MTV, true, 128>), grid, block, 0, stream, \
                           (const unsigned short*)wp.data_ptr(), (const unsigned short*)x.data_ptr(), \
                           nullptr, P.data_ptr<float>(), nullptr, (int)N, K, kc, nsplit); \
      else \
        hipLaunchKernelGGL((skinny_gemm_packed_kernel<MTV, true, 64>), grid, block, 0, stream, \
                           (const unsigned short*)wp.data_ptr(), (const unsigned short*)x.data_ptr(), \
                           nullptr, P.data_ptr<float>(), nullptr, (int)N, K, kc, nsplit); \
    } \
    break;
  if (nsplit == 1) {
    torch::Tensor P;
    switch (MT) { SGP_CASE(1) SGP_CASE(2) SGP_CASE(3) SGP_CASE(4) SGP_CASE(5) SGP_CASE(6) SGP_CASE(7) SGP_CASE(8) }
  } else {
    auto P = torch::empty({nsplit, M, (long long)N},
                          torch::TensorOptions().dtype(torch::kFloat32).device(x.device()));
    switch (MT) { SGP_CASE(1) SGP_CASE(2) SGP_CASE(3) SGP_CASE(4) SGP_CASE(5) SGP_CASE(6) SGP_CASE(7) SGP_CASE(8) }
    const long long MN = M * (long long)N;
    const int blocks = (int)std::min<long long>(2048, (MN / 4 + 255) / 256);
    hipLaunchKernelGGL(skinny_combine_kernel, dim3(blocks), dim3(256), 0, stream,
                       P.data_ptr<float>(), (unsigned short*)y.data_ptr(), bptr, MN, N, nsplit);
  }
#undef SGP_CASE
  return y;
}

// v3 (register-resident X) launcher — same contract as skinny_gemm_packed.
torch::Tensor skinny_gemm_packed_xreg(torch::Tensor x, torch::Tensor wp, int64_t N,
                                      c10::optional<torch::Tensor> bias) {
  CHK(x.is_cuda() && x.dtype() == torch::kBFloat16 && x.is_contiguous());
  CHK(wp.is_cuda() && wp.dtype() == torch::kBFloat16 && wp.is_contiguous());
  const long long K = wp.numel() / N;
  const long long M = x.numel() / K;
  CHK(M >= 32 && M <= 256 && M % 32 == 0);
  CHK(N % 128 == 0 && K % 64 == 0);
  const unsigned short* bptr = nullptr;
  if (bias.has_value()) {
    CHK(bias->is_contiguous() && bias->dtype() == torch::kBFloat16 && bias->numel() == N);
    bptr = (const unsigned short*)bias->data_ptr();
  }
  auto sizes = x.sizes().vec();
  sizes.back() = (long)N;
  auto y = torch::empty(sizes, x.options());
  const int ntiles = (int)(N / 128);
  int nsplit = 1;
  while (ntiles * nsplit < skinny_target_blocks() && (K / (nsplit * 2)) >= 1024 && nsplit < 16) nsplit *= 2;
  int kc = (int)((K / nsplit + 63) / 64 * 64);
  while ((long long)kc * (nsplit - 1) >= K) nsplit--;
  auto stream = cur_stream();
  const int MT = (int)(M / 32);
  const dim3 grid(ntiles * nsplit), block(256);
#define SGX_CASE(MTV) \
  case MTV: \
    if (nsplit == 1) { \
      hipLaunchKernelGGL((skinny_gemm_packed_xreg_kernel<MTV, false>), grid, block, 0, stream, \
                         (const unsigned short*)wp.data_ptr(), (const unsigned short*)x.data_ptr(), \
                         (unsigned short*)y.data_ptr(), nullptr, bptr, (int)N, K, kc, nsplit); \
    } else { \
      hipLaunchKernelGGL((skinny_gemm_packed_xreg_kernel<MTV, true>), grid, block, 0, stream, \
                         (const unsigned short*)wp.data_ptr(), (const unsigned short*)x.data_ptr(), \
                         nullptr, P.data_ptr<float>(), nullptr, (int)N, K, kc, nsplit); \
    } \
    break;
  if (nsplit == 1) {
    torch::Tensor P;
    switch (MT) { SGX_CASE(1) SGX_CASE(2) SGX_CASE(3) SGX_CASE(4) SGX_CASE(5) SGX_CASE(6) SGX_CASE(7) SGX_CASE(8) }
  } else {
    auto P = torch::empty({nsplit, M, (long long)N},
                          torch::TensorOptions().dtype(torch::kFloat32).device(x.device()));
    switch (MT) { SGX_CASE(1) SGX_CASE(2) SGX_CASE(3) SGX_CASE(4) SGX_CASE(5) SGX_CASE(6) SGX_CASE(7) SGX_CASE(8) }
    const long long MN = M * (long long)N;
    const int blocks = (int)std::min<long long>(2048, (MN / 4 + 255) / 256);
    hipLaunchKernelGGL(skinny_combine_kernel, dim3(blocks), dim3(256), 0, stream,
                       P.data_ptr<float>(), (unsigned short*)y.data_ptr(), bptr, MN, N, nsplit);
  }
#undef SGX_CASE
  return y;
}

// Fused SwiGLU + down-projection decode GEMM: gu is the [M, 2K] fused
// gate|up GEMM output, wp the prepacked down_proj ([N/32,K/16,64,8]);
// computes y = (silu(gate) * up) @ W_down^T with the activation applied in
// the X-staging — the intermediate [M, K] tensor never materializes.
torch::Tensor skinny_gemm_packed_swiglu(torch::Tensor gu, torch::Tensor wp, int64_t N,
                                        c10::optional<torch::Tensor> bias) {
  CHK(gu.is_cuda() && gu.dtype() == torch::kBFloat16 && gu.is_contiguous());
  CHK(wp.is_cuda() && wp.dtype() == torch::kBFloat16 && wp.is_contiguous());
  const long long K = wp.numel() / N;
  const long long M = gu.numel() / (2 * K);
  CHK(gu.size(-1) == 2 * K);
  CHK(M >= 32 && M <= 256 && M % 32 == 0);
  CHK(N % 128 == 0 && K % 64 == 0);
  const unsigned short* bptr = nullptr;
  if (bias.has_value()) {
    CHK(bias->is_contiguous() && bias->dtype() == torch::kBFloat16 && bias->numel() == N);
    bptr = (const unsigned short*)bias->data_ptr();
  }
  auto sizes = gu.sizes().vec();
  sizes.back() = (long)N;
  auto y = torch::empty(sizes, gu.options());
  const int ntiles = (int)(N / 128);
  int nsplit = 1;
  while (ntiles * nsplit < skinny_target_blocks() && (K / (nsplit * 2)) >= 1024 && nsplit < 16) nsplit *= 2;
  int kc = (int)((K / nsplit + 63) / 64 * 64);
  while ((long long)kc * (nsplit - 1) >= K) nsplit--;
  auto stream = cur_stream();
  const int MT = (int)(M / 32);
  const bool bk128 = (K % 128 == 0) && (kc % 128 == 0) && kc >= 2048
                     && getenv("XOT_SKINNY_BK64") == nullptr;
  const dim3 grid(ntiles * nsplit), block(256);
  const long long ldx = 2 * K;
#define SGS_CASE(MTV) \
  case MTV: \
    if (nsplit == 1) { \
      if (bk128) \
        hipLaunchKernelGGL((skinny_gemm_packed_kernel<MTV, false, 128, true>), grid, block, 0, stream, \
                           (const unsigned short*)wp.data_ptr(), (const unsigned short*)gu.data_ptr(), \
                           (unsigned short*)y.data_ptr(), nullptr, bptr, (int)N, K, kc, nsplit, ldx); \
      else \
        hipLaunchKernelGGL((skinny_gemm_packed_kernel<MTV, false, 64, true>), grid, block, 0, stream, \
                           (const unsigned short*)wp.data_ptr(), (const unsigned short*)gu.data_ptr(), \
                           (unsigned short*)y.data_ptr(), nullptr, bptr, (int)N, K, kc, nsplit, ldx); \
    } else { \
      if (bk128) \
        hipLaunchKernelGGL((skinny_gemm_packed_kernel<MTV, true, 128, true>), grid, block, 0, stream, \
                           (const unsigned short*)wp.data_ptr(), (const unsigned short*)gu.data_ptr(), \
                           nullptr, P.data_ptr<float>(), nullptr, (int)N, K, kc, nsplit, ldx); \
      else \
        hipLaunchKernelGGL((skinny_gemm_packed_kernel<MTV, true, 64, true>), grid, block, 0, stream, \
                           (const unsigned short*)wp.data_ptr(), (const unsigned short*)gu.data_ptr(), \
                           nullptr, P.data_ptr<float>(), nullptr, (int)N, K, kc, nsplit, ldx); \
    } \
    break;
  if (nsplit == 1) {
    torch::Tensor P;
    switch (MT) { SGS_CASE(1) SGS_CASE(2) SGS_CASE(3) SGS_CASE(4) SGS_CASE(5) SGS_CASE(6) SGS_CASE(7) SGS_CASE(8) }
  } else {
    auto P = torch::empty({nsplit, M, (long long)N},
                          torch::TensorOptions().dtype(torch::kFloat32).device(gu.device()));
    switch (MT) { SGS_CASE(1) SGS_CASE(2) SGS_CASE(3) SGS_CASE(4) SGS_CASE(5) SGS_CASE(6) SGS_CASE(7) SGS_CASE(8) }
    const long long MN = M * (long long)N;
    const int blocks = (int)std::min<long long>(2048, (MN / 4 + 255) / 256);
    hipLaunchKernelGGL(skinny_combine_kernel, dim3(blocks), dim3(256), 0, stream,
                       P.data_ptr<float>(), (unsigned short*)y.data_ptr(), bptr, MN, N, nsplit);
  }
#undef SGS_CASE
  return y;
}

// MoE grouped decode GEMM: x [E, C, K] (C = per-expert token capacity,
// 32..256, %32), wp: stacked prepacks [E, N/32, K/16, 64, 8] -> y [E, C, N].
// One launch for all experts (blockIdx.y = expert).
torch::Tensor skinny_gemm_grouped(torch::Tensor x, torch::Tensor wp, int64_t E, int64_t N) {
  CHK(x.is_cuda() && x.dtype() == torch::kBFloat16 && x.is_contiguous());
  CHK(wp.is_cuda() && wp.dtype() == torch::kBFloat16 && wp.is_contiguous());
  const long long K = wp.numel() / (E * N);
  const long long C = x.numel() / (K * E);
  CHK(C >= 32 && C <= 256 && C % 32 == 0);
  CHK(N % 128 == 0 && K % 64 == 0 && E >= 1 && E <= 256);
  auto y = torch::empty({(long)E, (long)C, (long)N}, x.options());
  const int ntiles = (int)(N / 128);
  int nsplit = 1;
  while (ntiles * nsplit * E < skinny_target_blocks() && (K / (nsplit * 2)) >= 1024 && nsplit < 16) nsplit *= 2;
  int kc = (int)((K / nsplit + 63) / 64 * 64);
  while ((long long)kc * (nsplit - 1) >= K) nsplit--;
  auto stream = cur_stream();
  const int MT = (int)(C / 32);
  const dim3 grid(ntiles * nsplit, (unsigned)E), block(256);
  const bool bk128 = (K % 128 == 0) && (kc % 128 == 0) && kc >= 2048
                     && getenv("XOT_SKINNY_BK64") == nullptr;
#define SGG_CASE(MTV) \
  case MTV: \
    if (nsplit == 1) { \
      if (bk128) \
        hipLaunchKernelGGL((skinny_gemm_packed_kernel<MTV, false, 128>), grid, block, 0, stream, \
                           (const unsigned short*)wp.data_ptr(), (const unsigned short*)x.data_ptr(), \
                           (unsigned short*)y.data_ptr(), nullptr, nullptr, (int)N, K, kc, nsplit); \
      else \
        hipLaunchKernelGGL((skinny_gemm_packed_kernel<MTV, false, 64>), grid, block, 0, stream, \
                           (const unsigned short*)wp.data_ptr(), (const unsigned short*)x.data_ptr(), \
                           (unsigned short*)y.data_ptr(), nullptr, nullptr, (int)N, K, kc, nsplit); \
    } else { \
      if (bk128) \
        hipLaunchKernelGGL((skinny_gemm_packed_kernel<MTV, true, 128>), grid, block, 0, stream, \
                           (const unsigned short*)wp.data_ptr(), (const unsigned short*)x.data_ptr(), \
                           nullptr, P.data_ptr<float>(), nullptr, (int)N, K, kc, nsplit); \
      else \
        hipLaunchKernelGGL((skinny_gemm_packed_kernel<MTV, true, 64>), grid, block, 0, stream, \
                           (const unsigned short*)wp.data_ptr(), (const unsigned short*)x.data_ptr(), \
                           nullptr, P.data_ptr<float>(), nullptr, (int)N, K, kc, nsplit); \
    } \
    break;
  if (nsplit == 1) {
    torch::Tensor P;
    switch (MT) { SGG_CASE(1) SGG_CASE(2) SGG_CASE(3) SGG_CASE(4) SGG_CASE(5) SGG_CASE(6) SGG_CASE(7) SGG_CASE(8) }
  } else {
    auto P = torch::empty({nsplit, (long)(E * C), (long)N},
                          torch::TensorOptions().dtype(torch::kFloat32).device(x.device()));
    switch (MT) { SGG_CASE(1) SGG_CASE(2) SGG_CASE(3) SGG_CASE(4) SGG_CASE(5) SGG_CASE(6) SGG_CASE(7) SGG_CASE(8) }
    const long long MN = E * C * N;
    const int blocks = (int)std::min<long long>(2048, (MN / 4 + 255) / 256);
    hipLaunchKernelGGL(skinny_combine_kernel, dim3(blocks), dim3(256), 0, stream,
                       P.data_ptr<float>(), (unsigned short*)y.data_ptr(), nullptr, MN, N, nsplit);
  }
#undef SGG_CASE
  return y;
}

// x: [M, K] bf16 -> (x8 uint8 [M, K], s_x fp32 [M])
std::vector<torch::Tensor> quant_fp8_rows(torch::Tensor x) {
  CHK(x.is_cuda() && x.dtype() == torch::kBFloat16 && x.is_contiguous());
  const long long K = x.size(-1);
  const long long M = x.numel() / K;
  CHK(K % 8 == 0);
  auto x8 = torch::empty({M, K}, torch::TensorOptions().dtype(torch::kUInt8).device(x.device()));
  auto sx = torch::empty({M}, torch::TensorOptions().dtype(torch::kFloat32).device(x.device()));
  hipLaunchKernelGGL(quant_fp8_rows_kernel, dim3((unsigned)M), dim3(256), 0, cur_stream(),
                     (const unsigned short*)x.data_ptr(), (unsigned char*)x8.data_ptr(),
                     sx.data_ptr<float>(), K);
  return {x8, sx};
}

// W8A8 e4m3 decode GEMM. x8/sx from quant_fp8_rows; wp8: fp8 prepack
// [E][N/32][K/16][64][8] bytes; sw: [E, N] fp32 per-channel scales. E == 1
// for plain GEMMs; E > 1 = MoE grouped mode (x8 is [E, C, K]).
torch::Tensor skinny_gemm_fp8(torch::Tensor x8, torch::Tensor sx, torch::Tensor wp8,
                              torch::Tensor sw, int64_t E, int64_t N,
                              c10::optional<torch::Tensor> bias) {
  CHK(x8.is_cuda() && x8.dtype() == torch::kUInt8 && x8.is_contiguous());
  CHK(wp8.is_cuda() && wp8.dtype() == torch::kUInt8 && wp8.is_contiguous());
  CHK(sx.dtype() == torch::kFloat32 && sw.dtype() == torch::kFloat32);
  CHK(sw.is_contiguous() && sx.is_contiguous());
  const long long K = wp8.numel() / (E * N);
  const long long M = x8.numel() / (K * E);  // rows per expert
  CHK(M >= 32 && M <= 256 && M % 32 == 0);
  CHK(N % 128 == 0 && K % 64 == 0 && sw.numel() == E * N && sx.numel() == E * M);
  const unsigned short* bptr = nullptr;
  if (bias.has_value()) {
    CHK(bias->is_contiguous() && bias->dtype() == torch::kBFloat16 && bias->numel() == N);
    bptr = (const unsigned short*)bias->data_ptr();
  }
  auto y = torch::empty({(long)(E * M), (long)N},
                        torch::TensorOptions().dtype(torch::kBFloat16).device(x8.device()));
  const int ntiles = (int)(N / 128);
  int nsplit = 1;
  while (ntiles * nsplit * E < skinny_target_blocks() && (K / (nsplit * 2)) >= 1024 && nsplit < 16) nsplit *= 2;
  int kc = (int)((K / nsplit + 63) / 64 * 64);
  while ((long long)kc * (nsplit - 1) >= K) nsplit--;
  auto stream = cur_stream();
  const int MT = (int)(M / 32);
  const dim3 grid(ntiles * nsplit, (unsigned)E), block(256);
#define SGF_CASE(MTV) \
  case MTV: \
    if (nsplit == 1) { \
      hipLaunchKernelGGL((skinny_gemm_fp8_kernel<MTV, false>), grid, block, 0, stream, \
                         (const unsigned char*)wp8.data_ptr(), (const unsigned char*)x8.data_ptr(), \
                         sw.data_ptr<float>(), sx.data_ptr<float>(), \
                         (unsigned short*)y.data_ptr(), nullptr, bptr, (int)N, K, kc, nsplit); \
    } else { \
      hipLaunchKernelGGL((skinny_gemm_fp8_kernel<MTV, true>), grid, block, 0, stream, \
                         (const unsigned char*)wp8.data_ptr(), (const unsigned char*)x8.data_ptr(), \
                         sw.data_ptr<float>(), sx.data_ptr<float>(), \
                         nullptr, P.data_ptr<float>(), nullptr, (int)N, K, kc, nsplit); \
    } \
    break;
  if (nsplit == 1) {
    torch::Tensor P;
    switch (MT) { SGF_CASE(1) SGF_CASE(2) SGF_CASE(3) SGF_CASE(4) SGF_CASE(5) SGF_CASE(6) SGF_CASE(7) SGF_CASE(8) }
  } else {
    auto P = torch::empty({nsplit, (long)(E * M), (long)N},
                          torch::TensorOptions().dtype(torch::kFloat32).device(x8.device()));
    switch (MT) { SGF_CASE(1) SGF_CASE(2) SGF_CASE(3) SGF_CASE(4) SGF_CASE(5) SGF_CASE(6) SGF_CASE(7) SGF_CASE(8) }
    const long long MN = E * M * N;
    const int blocks = (int)std::min<long long>(2048, (MN / 4 + 255) / 256);
    hipLaunchKernelGGL(skinny_combine_kernel, dim3(blocks), dim3(256), 0, stream,
                       P.data_ptr<float>(), (unsigned short*)y.data_ptr(), bptr, MN, N, nsplit);
  }
#undef SGF_CASE
  return y;
}

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.def("quant_fp8_rows", &quant_fp8_rows, "per-row dynamic e4m3 quantization");
  m.def("skinny_gemm_fp8", &skinny_gemm_fp8,
        "W8A8 e4m3 decode GEMM on prepacked weights (per-channel/per-token scales)",
        py::arg("x8"), py::arg("sx"), py::arg("wp8"), py::arg("sw"), py::arg("n_experts"),
        py::arg("n"), py::arg("bias") = py::none());
  m.def("skinny_gemm", &skinny_gemm, "decode GEMM y = x @ w^T (+bias), bf16 MFMA weight-streaming",
        py::arg("x"), py::arg("w"), py::arg("bias") = py::none());
  m.def("skinny_gemm_packed_xreg", &skinny_gemm_packed_xreg,
        "decode GEMM on prepacked weights, register-resident X (M=128/256 shapes)",
        py::arg("x"), py::arg("wp"), py::arg("N"), py::arg("bias") = py::none());
  m.def("skinny_gemm_packed_swiglu", &skinny_gemm_packed_swiglu,
        "fused silu(gate)*up + down-proj decode GEMM on the prepacked weight",
        py::arg("gu"), py::arg("wp"), py::arg("n"), py::arg("bias") = py::none());
  m.def("skinny_gemm_packed", &skinny_gemm_packed,
        "decode GEMM on prepacked weights (MFMA fragment order)",
        py::arg("x"), py::arg("wp"), py::arg("n"), py::arg("bias") = py::none());
  m.def("skinny_gemm_grouped", &skinny_gemm_grouped,
        "MoE grouped decode GEMM on stacked prepacked expert weights",
        py::arg("x"), py::arg("wp"), py::arg("n_experts"), py::arg("n"));
  m.def("swiglu_packed", &swiglu_packed, "SwiGLU on the packed [gate|up] GEMM output");
  m.def("geglu_packed", &geglu_packed, "GeGLU (tanh gelu) on the packed [gate|up] GEMM output");
  m.def("rmsnorm", &rmsnorm, "RMSNorm (bf16, CDNA4); w_bias=1 gives gemma-style (1+w)",
        py::arg("x"), py::arg("w"), py::arg("eps"), py::arg("w_bias") = 0.0);
  m.def("rmsnorm_residual", &rmsnorm_residual, "fused residual add + RMSNorm",
        py::arg("x"), py::arg("res"), py::arg("w"), py::arg("eps"), py::arg("w_bias") = 0.0);
  m.def("rope_qkv_append", &rope_qkv_append,
        "fused (qk-RMSNorm +) RoPE + KV-cache append on packed qkv",
        py::arg("qkv"), py::arg("cos"), py::arg("sin"), py::arg("positions"), py::arg("kc"),
        py::arg("vc"), py::arg("n_heads"), py::arg("n_kv_heads"), py::arg("head_dim"),
        py::arg("kp") = py::none(), py::arg("vp") = py::none(),
        py::arg("q_norm") = py::none(), py::arg("k_norm") = py::none(),
        py::arg("norm_eps") = 1e-6,
        py::arg("k_scale") = py::none(), py::arg("v_scale") = py::none());
  m.def("attn_decode", &attn_decode, "GQA decode attention (flash-decoding split-KV)");
  m.def("attn_decode_mfma", &attn_decode_mfma,
        "GQA decode attention on matrix cores (packed cache, hd=128); "
        "softcap/window: gemma2 logit soft-capping and sliding window",
        py::arg("q"), py::arg("kp"), py::arg("vp"), py::arg("seq_lens"), py::arg("t_capacity"),
        py::arg("scale") = 0.0, py::arg("softcap") = 0.0, py::arg("window") = 0,
        py::arg("k_scale") = py::none(), py::arg("v_scale") = py::none());
  m.def("attn_prefill_mfma", &attn_prefill_mfma,
        "causal GQA prefill flash attention on matrix cores (packed cache, hd=128)",
        py::arg("q"), py::arg("kp"), py::arg("vp"), py::arg("start_pos"),
        py::arg("scale") = 0.0, py::arg("softcap") = 0.0, py::arg("window") = 0);
  m.def("moe_route", &moe_route,
        "fused MoE router: softmax-topk (mode 0) / sigmoid+group-limited (mode 1)",
        py::arg("logits"), py::arg("bias") = py::none(), py::arg("k") = 2,
        py::arg("mode") = 0, py::arg("n_group") = 1, py::arg("topk_group") = 1,
        py::arg("routed_scale") = 1.0, py::arg("norm_topk") = false);
  m.def("moe_build", &moe_build,
        "MoE decode routing: counting-sort token-expert pairs to padded per-expert slots");
  m.def("moe_combine", &moe_combine,
        "MoE decode combine: out[t] = sum_j w[t,j] * y[pos(t,j)] (deterministic)");
  m.def("mla_q_prep", &mla_q_prep,
        "MLA absorbed-query finisher: rope the 64-dim tail + assemble [B,H,576]; "
        "fp8=True returns (q8, per-head scales)",
        py::arg("q"), py::arg("q_lat"), py::arg("cos"), py::arg("sin"), py::arg("positions"),
        py::arg("nope"), py::arg("interleave") = false, py::arg("fp8") = false);
  m.def("mla_prep_append", &mla_prep_append,
        "fused MLA kv prep: latent RMSNorm + shared-key rope + both cache layouts",
        py::arg("ckv"), py::arg("w"), py::arg("cos"), py::arg("sin"), py::arg("positions"),
        py::arg("lat_c"), py::arg("rot_c"), py::arg("kp"), py::arg("vp"), py::arg("eps"),
        py::arg("interleave") = false, py::arg("k_scale") = py::none());
  m.def("mla_append", &mla_append,
        "append MLA latent+rope token stream into the fragment-packed cache");
  m.def("attn_decode_mla", &attn_decode_mla,
        "MLA decode attention (absorbed latent MQA) on matrix cores; fp8 cache mode",
        py::arg("q"), py::arg("kp"), py::arg("vp"), py::arg("seq_lens"),
        py::arg("scale") = 0.0, py::arg("q_scale") = py::none(), py::arg("k_scale") = py::none());
  m.def("mfma16_probe", &mfma16_probe, "v_mfma_f32_16x16x32_bf16 layout probe (tests)");
  m.def("swiglu", &swiglu, "SwiGLU activation");
}
