// Matrix-core form of the windowed sink attention for 16-bit prompts
// (attn_window.hip states the semantics and covers every other shape).
//
// One workgroup = 64 queries of one head, 4 waves x 16 query rows, key
// tiles of 64 from the window's first key on.  Both key parts are staged
// side by side in LDS (16 B row pad), values transposed (Vt[d][key], XOR
// swizzled in 16-byte blocks so that the packed two-key writes and the
// fragment reads both spread over the banks).  Queries are staged and
// rotated once.  Scores and the online softmax stay in fp32 registers; the
// sink starts the running maximum and denominator, so a row is never
// empty.  The epilogue applies 1/l and the output gate.
#include "seq_common.h"

namespace {

constexpr int TPB = 256;
constexpr int BM = 64, BN = 64;

struct PArgs {
  const bf16_t *q, *k1, *k2, *v, *g;
  u64 k1_ld, k2_ld, v_ld, ldg;
  const i32* own_row;
  const float *inv_freq, *sink;
  bf16_t* out;
  int heads, d1, d2, rot_dims, dv, window;
  float scale;
  int group, cap;        // query heads a key/value head; cache rows a slot
  u64 ldo;
  float gain;
};

__device__ __forceinline__ u32 swz(u32 row) { return (row ^ (row >> 3)) & 7; }

template <int KS, int VT>
__global__ __launch_bounds__(TPB) void attn_window_prompt_mfma(SeqView sv,
                                                               PArgs A) {
  constexpr int QKP = KS * 32, VP = VT * 16;
  constexpr int KROW = QKP * 2 + 16, PROW = BN * 2 + 16;
  extern __shared__ __attribute__((aligned(16))) char smem[];
  char* ldsK = smem;
  char* ldsV = ldsK + BN * KROW;
  char* ldsP = ldsV + VP * 128;
  // the last queries see the most keys: they start first
  const int q0 = (gridDim.x - 1 - blockIdx.x) * BM;
  const int s = blockIdx.z, h = blockIdx.y, kh = h / A.group;
  const int row0 = sv.cu[s], cnt = sv.cu[s + 1] - row0;
  if (q0 >= cnt) return;
  const int slot = sv.slots[s], len0 = sv.lens[slot];
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  const int l15 = lane & 15, l4 = lane >> 4;
  const int D = A.d1 + A.d2;

  // ---- queries: stage, rotate the second part, keep as A-fragments ----
  for (int c = tid; c < BM * (QKP / 8); c += TPB) {
    const int r = c / (QKP / 8), e0 = (c % (QKP / 8)) * 8;
    u32x4 d = {0, 0, 0, 0};
    if (q0 + r < cnt && e0 < D)
      d = *(const u32x4*)(A.q + ((u64)(row0 + q0 + r) * A.heads + h) * D + e0);
    *(u32x4*)(ldsK + r * KROW + e0 * 2) = d;
  }
  __syncthreads();
  const int half = A.rot_dims / 2;
  for (int c = tid; c < BM * half; c += TPB) {
    const int r = c / half, j = c % half;
    unsigned short* p = (unsigned short*)(ldsK + r * KROW) + A.d1 + j;
    float sn, cs;
    sincosf((float)(len0 + q0 + r) * A.inv_freq[j], &sn, &cs);
    const float u = bf16_bits_to_f32(p[0]), w = bf16_bits_to_f32(p[half]);
    p[0] = (unsigned short)f32_to_bf16_bits_rne(u * cs - w * sn);
    p[half] = (unsigned short)f32_to_bf16_bits_rne(w * cs + u * sn);
  }
  __syncthreads();
  s16x8 qf[KS];
#pragma unroll
  for (int ks = 0; ks < KS; ++ks)
    qf[ks] = *(const s16x8*)(ldsK + (wave * 16 + l15) * KROW +
                             (ks * 32 + l4 * 8) * 2);

  const float snk = A.sink[h];
  float mrun[4] = {snk, snk, snk, snk};
  float lrun[4] = {1.f, 1.f, 1.f, 1.f};
  f32x4 oacc[VT] = {};

  const int p_lo = len0 + q0, p_hi = len0 + min(q0 + BM, cnt) - 1;
  const int lo = p_lo < A.window ? 0 : p_lo - A.window + 1, hi = p_hi + 1;
  // row of key 0: in the step's key buffer, or in the cache
  const long base = A.own_row != nullptr ? (long)A.own_row[s] - len0
                                         : (long)slot * A.cap;
  for (int t0 = lo; t0 < hi; t0 += BN) {
    __syncthreads();
#pragma unroll 4
    for (int c = tid; c < BN * (QKP / 8); c += TPB) {
      const int key = c / (QKP / 8), e0 = (c % (QKP / 8)) * 8;
      const u64 kr = (u64)(base + min(t0 + key, hi - 1));
      u32x4 d = {0, 0, 0, 0};
      if (e0 < A.d1)
        d = *(const u32x4*)(A.k1 + kr * A.k1_ld + kh * A.d1 + e0);
      else if (e0 < D)
        d = *(const u32x4*)(A.k2 + kr * A.k2_ld + (e0 - A.d1));
      *(u32x4*)(ldsK + key * KROW + e0 * 2) = d;
    }
#pragma unroll 2
    for (int c = tid; c < (BN / 2) * (VP / 8); c += TPB) {
      const int kp = c / (VP / 8), dg = c % (VP / 8);
      u32x4 a = {0, 0, 0, 0}, b = {0, 0, 0, 0};
      if (dg * 8 < A.dv) {
        const u64 ra = (u64)(base + min(t0 + 2 * kp, hi - 1));
        const u64 rb = (u64)(base + min(t0 + 2 * kp + 1, hi - 1));
        a = *(const u32x4*)(A.v + ra * A.v_ld + kh * A.dv + dg * 8);
        b = *(const u32x4*)(A.v + rb * A.v_ld + kh * A.dv + dg * 8);
      }
      const u32 blk = kp >> 2, off = (kp & 3) * 4;
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        const u32 x = (a[e >> 1] >> ((e & 1) * 16)) & 0xFFFFu;
        const u32 y = (b[e >> 1] >> ((e & 1) * 16)) & 0xFFFFu;
        const u32 d = dg * 8 + e;
        *(u32*)(ldsV + d * 128 + ((blk ^ swz(d)) << 4) + off) = x | (y << 16);
      }
    }
    __syncthreads();

    f32x4 sc[BN / 16] = {};
#pragma unroll
    for (int ks = 0; ks < KS; ++ks)
#pragma unroll
      for (int nt = 0; nt < BN / 16; ++nt) {
        const s16x8 kf = *(const s16x8*)(ldsK + (nt * 16 + l15) * KROW +
                                         (ks * 32 + l4 * 8) * 2);
        sc[nt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(qf[ks], kf, sc[nt],
                                                         0, 0, 0);
      }
#pragma unroll
    for (int nt = 0; nt < BN / 16; ++nt) {
      const int j = t0 + nt * 16 + l15;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int pos = p_lo + wave * 16 + l4 * 4 + r;
        const bool ok = j <= pos && pos - j < A.window && j < hi;
        sc[nt][r] = ok ? sc[nt][r] * A.scale : -INFINITY;
      }
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      float mx = fmaxf(fmaxf(sc[0][r], sc[1][r]), fmaxf(sc[2][r], sc[3][r]));
#pragma unroll
      for (int o = 8; o > 0; o >>= 1) mx = fmaxf(mx, __shfl_xor(mx, o, 64));
      const float mn = fmaxf(mrun[r], mx);
      const float al = __expf(mrun[r] - mn);
      float ps = 0.f;
#pragma unroll
      for (int nt = 0; nt < BN / 16; ++nt) {
        const float p = __expf(sc[nt][r] - mn);
        sc[nt][r] = p;
        ps += p;
      }
#pragma unroll
      for (int o = 8; o > 0; o >>= 1) ps += __shfl_xor(ps, o, 64);
      lrun[r] = lrun[r] * al + ps;
      mrun[r] = mn;
#pragma unroll
      for (int on = 0; on < VT; ++on) oacc[on][r] *= al;
    }
    // P to A-fragment layout through this wave's own LDS slab
    char* pw = ldsP + wave * 16 * PROW;
#pragma unroll
    for (int nt = 0; nt < BN / 16; ++nt)
#pragma unroll
      for (int r = 0; r < 4; ++r)
        *(unsigned short*)(pw + (l4 * 4 + r) * PROW + (nt * 16 + l15) * 2) =
            (unsigned short)f32_to_bf16_bits_rne(sc[nt][r]);
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
#pragma unroll
    for (int k2 = 0; k2 < BN / 32; ++k2) {
      const s16x8 pf =
          *(const s16x8*)(pw + l15 * PROW + (k2 * 32 + l4 * 8) * 2);
#pragma unroll
      for (int on = 0; on < VT; ++on) {
        const u32 d = on * 16 + l15, blk = k2 * 4 + l4;
        const s16x8 vf =
            *(const s16x8*)(ldsV + d * 128 + ((blk ^ swz(d)) << 4));
        oacc[on] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(pf, vf, oacc[on],
                                                           0, 0, 0);
      }
    }
  }

#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int qr = q0 + wave * 16 + l4 * 4 + r;
    if (qr >= cnt) continue;
    const float inv = A.gain / lrun[r];
    const u64 row = row0 + qr;
    const bf16_t* gr = A.g + row * A.ldg + h * A.dv;
    bf16_t* o = A.out + row * A.ldo + h * A.dv;
#pragma unroll
    for (int on = 0; on < VT; ++on) {
      const int e = on * 16 + l15;
      if (e < A.dv)
        stf(o + e, oacc[on][r] * inv *
                       (A.g != nullptr ? sigmoid_f(ldf(gr + e)) : 1.f));
    }
  }
}

template <int KS, int VT>
hipError_t launch(const SeqView& sv, const PArgs& A, int max_count,
                  hipStream_t stream) {
  constexpr size_t lds = (size_t)BN * (KS * 64 + 16) + VT * 16 * 128 +
                         4 * 16 * (BN * 2 + 16);
  static bool set = false;
  if (!set && lds > 64 * 1024) {
    LFMQ_CHECK_HIP(hipFuncSetAttribute(
        (const void*)attn_window_prompt_mfma<KS, VT>,
        hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds));
    set = true;
  }
  hipLaunchKernelGGL((attn_window_prompt_mfma<KS, VT>),
                     dim3((max_count + BM - 1) / BM, A.heads, sv.b),
                     dim3(TPB), lds, stream, sv, A);
  return hipGetLastError();
}

hipError_t dispatch(const SeqView& sv, const PArgs& A, int max_count,
                    hipStream_t stream) {
  const int ks = (A.d1 + A.d2 + 31) / 32, vt = (A.dv + 15) / 16;
#define GO(K, V) return launch<K, V>(sv, A, max_count, stream)
#define GOV(K)                                                               \
  do {                                                                       \
    if (vt <= 4) GO(K, 4);                                                   \
    if (vt <= 8) GO(K, 8);                                                   \
    GO(K, 16);                                                               \
  } while (0)
  if (ks <= 2) GOV(2);
  if (ks <= 4) GOV(4);
  if (ks <= 6) GOV(6);
  GOV(8);
#undef GOV
#undef GO
}

bool al16(const void* p) { return ((u64)p & 15) == 0; }

}  // namespace

// false: this shape belongs to the general kernel
bool lfmq_attn_window_prompt_mfma_ok(const void* q, const void* k1,
                                     long k1_ld, const void* k2, long k2_ld,
                                     const void* v, long v_ld, int d1, int d2,
                                     int dv) {
  return d1 % 8 == 0 && d2 % 8 == 0 && dv % 8 == 0 && k1_ld % 8 == 0 &&
         k2_ld % 8 == 0 && v_ld % 8 == 0 && d1 + d2 <= 256 && dv <= 256 &&
         al16(q) && al16(k1) && al16(k2) && al16(v);
}

hipError_t lfmq_attn_window_prompt_mfma(
    const void* q, const void* k1, long k1_ld, const void* k2, long k2_ld,
    const void* v, long v_ld, const SeqView& sv, const void* own_row,
    const void* inv_freq, const void* sink, const void* g, long ldg,
    void* out, int heads, int d1, int d2, int rot_dims, int dv, int window,
    float scale, int max_count, hipStream_t stream) {
  PArgs A{(const bf16_t*)q, (const bf16_t*)k1, (const bf16_t*)k2,
          (const bf16_t*)v, (const bf16_t*)g, (u64)k1_ld, (u64)k2_ld,
          (u64)v_ld, (u64)ldg, (const i32*)own_row, (const float*)inv_freq,
          (const float*)sink, (bf16_t*)out, heads, d1, d2, rot_dims, dv,
          window, scale, 1, 0, (u64)heads * dv, 1.f};
  return dispatch(sv, A, max_count, stream);
}

// grouped queries over a key/value cache (attn_window.hip:
// lfmq_attn_grouped)
bool lfmq_attn_grouped_mfma_ok(const void* q, const void* kc, const void* vc,
                               int dim, int dv) {
  return dim % 8 == 0 && dv % 8 == 0 && dim <= 256 && dv <= 256 && al16(q) &&
         al16(kc) && al16(vc);
}

hipError_t lfmq_attn_grouped_mfma(const void* q, const void* kc,
                                  const void* vc, const SeqView& sv,
                                  const void* sink, void* out, long ldo,
                                  int heads, int group, int dim, int dv,
                                  int cap, float scale, float gain,
                                  int max_count, hipStream_t stream) {
  const u64 kv = heads / group;
  PArgs A{(const bf16_t*)q, (const bf16_t*)kc, (const bf16_t*)kc,
          (const bf16_t*)vc, nullptr, kv * dim, 0, kv * dv, 0, nullptr,
          nullptr, (const float*)sink, (bf16_t*)out, heads, dim, 0, 0, dv,
          INT32_MAX, scale, group, cap, (u64)ldo, gain};
  return dispatch(sv, A, max_count, stream);
}
