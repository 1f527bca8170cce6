// Matrix-core decode attention over the latent ring cache (one token per
// sequence, absorbed queries; attn_window.hip states the semantics and
// covers every other shape).
//
// All heads share the latent row {c, k_rot}: the heads of a group are the
// M rows of the products, so one pass over the window's rows serves 16 or
// 32 heads.  A workgroup = one key range x one head group, 4 waves, tiles
// of 32 keys.  A tile is loaded once (the next one is in flight while this
// one is multiplied) and staged twice: row-major for the scores, and c
// transposed (80-byte rows: packed two-key writes and fragment reads both
// spread over the banks) for the weighted sum.  Queries stay in registers;
// scores, softmax and sums in fp32.  Emits {sum p c, max, sum p}.
#include "seq_common.h"

namespace {

constexpr int TPB = 256;
constexpr int KT = 32;
constexpr int VROW = 80;

struct LArgs {
  const bf16_t *q, *ring;
  float* part;
  int heads, rank, rot, window, cap, splits;
  float scale;
};

template <int KS>
constexpr int krow() { return KS * 64 + 16; }

template <int KS, int NT, int MT>
constexpr size_t lds_bytes() {
  return (size_t)KT * krow<KS>() + (size_t)NT * 64 * VROW +
         (size_t)MT * 16 * (KT * 2 + 16) + (size_t)MT * 16 * (KT + 1) * 4 +
         MT * 16 * 4;
}

template <int KS, int NT, int MT>
__global__ __launch_bounds__(TPB) void attn_latent_decode_mfma(SeqView sv,
                                                               LArgs A) {
  constexpr int KROW = krow<KS>(), HG = MT * 16, PROW = KT * 2 + 16;
  constexpr int CG = KS * 4;                  // 16-byte columns of a row
  constexpr int NI = (CG * 16 + TPB - 1) / TPB;
  extern __shared__ __attribute__((aligned(16))) char smem[];
  char* ldsK = smem;
  char* ldsV = ldsK + KT * KROW;
  char* ldsP = ldsV + NT * 64 * VROW;
  float* ldsS = (float*)(ldsP + HG * PROW);   // [HG][KT + 1]
  float* ldsA = ldsS + HG * (KT + 1);         // rescale per head
  const int s = blockIdx.z, h0 = blockIdx.y * HG;
  const int slot = sv.slots[s];
  const int pos = sv.lens[slot];
  const int D = A.rank + A.rot;
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  const int l15 = lane & 15, l4 = lane >> 4;

  int lo = max(0, pos - A.window + 1);
  const int per = ((pos + 1 - lo + A.splits - 1) / A.splits + KT - 1) / KT * KT;
  lo += blockIdx.x * per;
  const int hi = min(pos + 1, lo + per);
  const bf16_t* ring = A.ring + (u64)slot * A.cap * D;

  // score role: head tile qm, key tile qn
  const int qm = MT == 2 ? (wave & 1) : 0, qn = MT == 2 ? (wave >> 1) : wave;
  const bool scores = qn < KT / 16;
  s16x8 qf[KS];
  {
    const int h = h0 + qm * 16 + l15;
    const bf16_t* qr = A.q + ((u64)s * A.heads + h) * D;
    const s16x8 z = {0, 0, 0, 0, 0, 0, 0, 0};
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
      const int k = ks * 32 + l4 * 8;
      qf[ks] = (scores && h < A.heads && k < D) ? *(const s16x8*)(qr + k) : z;
    }
  }
  f32x4 acc[MT][NT] = {};
  // softmax role: 8 threads a head row (HG * 8 <= 256), 4 keys each
  const int sr = tid >> 3, sp = tid & 7;
  float m = -INFINITY, l = 0.f;

  u32x4 xa[NI], xb[NI];
  auto fetch = [&](int t0) {
#pragma unroll
    for (int i = 0; i < NI; ++i) {
      const int it = i * TPB + tid;
      const int kp = it & 15, e0 = (it >> 4) * 8;
      const u32x4 z = {0, 0, 0, 0};
      const int ja = t0 + 2 * kp, jb = ja + 1;
      const bool c = e0 < D;
      xa[i] = (c && ja < hi) ? *(const u32x4*)(ring + (u64)(ja % A.cap) * D + e0)
                             : z;
      xb[i] = (c && jb < hi) ? *(const u32x4*)(ring + (u64)(jb % A.cap) * D + e0)
                             : z;
    }
  };
  if (lo < hi) fetch(lo);
  for (int t0 = lo; t0 < hi; t0 += KT) {
    __syncthreads();                 // the last tile is consumed
#pragma unroll
    for (int i = 0; i < NI; ++i) {
      const int it = i * TPB + tid;
      const int kp = it & 15, cg = it >> 4;
      if (cg >= CG) break;
      *(u32x4*)(ldsK + (2 * kp) * KROW + cg * 16) = xa[i];
      *(u32x4*)(ldsK + (2 * kp + 1) * KROW + cg * 16) = xb[i];
      if (cg * 8 < A.rank) {
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          const u32 sh = (e & 1) * 16;
          *(u32*)(ldsV + (cg * 8 + e) * VROW + kp * 4) =
              ((xa[i][e >> 1] >> sh) & 0xFFFFu) |
              (((xb[i][e >> 1] >> sh) & 0xFFFFu) << 16);
        }
      }
    }
    if (t0 + KT < hi) fetch(t0 + KT);
    __syncthreads();
    if (scores) {
      f32x4 c = {};
#pragma unroll
      for (int ks = 0; ks < KS; ++ks) {
        const s16x8 kf = *(const s16x8*)(ldsK + (qn * 16 + l15) * KROW +
                                         (ks * 32 + l4 * 8) * 2);
        c = __builtin_amdgcn_mfma_f32_16x16x32_bf16(qf[ks], kf, c, 0, 0, 0);
      }
#pragma unroll
      for (int r = 0; r < 4; ++r)
        ldsS[(qm * 16 + l4 * 4 + r) * (KT + 1) + qn * 16 + l15] =
            t0 + qn * 16 + l15 < hi ? c[r] * A.scale : -INFINITY;
    }
    __syncthreads();
    if (sr < HG) {
      float x[4], mx = -INFINITY;
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        x[i] = ldsS[sr * (KT + 1) + sp * 4 + i];
        mx = fmaxf(mx, x[i]);
      }
#pragma unroll
      for (int o = 4; o > 0; o >>= 1) mx = fmaxf(mx, __shfl_xor(mx, o, 64));
      const float mn = fmaxf(m, mx);           // a tile has a visible key
      const float al = __expf(m - mn);
      float sum = 0.f;
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        x[i] = __expf(x[i] - mn);
        sum += x[i];
      }
#pragma unroll
      for (int o = 4; o > 0; o >>= 1) sum += __shfl_xor(sum, o, 64);
      l = l * al + sum;
      m = mn;
      *(u32x2*)(ldsP + sr * PROW + sp * 8) =
          u32x2{pack_bf16x2(x[0], x[1]), pack_bf16x2(x[2], x[3])};
      if (sp == 0) ldsA[sr] = al;
    }
    __syncthreads();
    s16x8 pf[MT];
#pragma unroll
    for (int mt = 0; mt < MT; ++mt) {
      pf[mt] = *(const s16x8*)(ldsP + (mt * 16 + l15) * PROW + l4 * 16);
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const float al = ldsA[mt * 16 + l4 * 4 + r];
#pragma unroll
        for (int j = 0; j < NT; ++j) acc[mt][j][r] *= al;
      }
    }
#pragma unroll
    for (int j = 0; j < NT; ++j) {
      const s16x8 vf = *(const s16x8*)(
          ldsV + ((wave * NT + j) * 16 + l15) * VROW + l4 * 16);
#pragma unroll
      for (int mt = 0; mt < MT; ++mt)
        acc[mt][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
            pf[mt], vf, acc[mt][j], 0, 0, 0);
    }
  }

  const u64 pr = A.rank + 2;
  float* out = A.part + ((u64)s * A.splits + blockIdx.x) * A.heads * pr;
#pragma unroll
  for (int mt = 0; mt < MT; ++mt)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int h = h0 + mt * 16 + l4 * 4 + r;
      if (h >= A.heads) continue;
#pragma unroll
      for (int j = 0; j < NT; ++j) {
        const int e = (wave * NT + j) * 16 + l15;
        if (e < A.rank) out[h * pr + e] = acc[mt][j][r];
      }
    }
  if (sr < HG && sp == 0 && h0 + sr < A.heads) {
    out[(h0 + sr) * pr + A.rank] = m;
    out[(h0 + sr) * pr + A.rank + 1] = l;
  }
}

template <int KS, int NT, int MT>
hipError_t launch(const SeqView& sv, const LArgs& A, hipStream_t stream) {
  constexpr size_t lds = lds_bytes<KS, NT, MT>();
  static bool set = false;
  if (!set && lds > 64 * 1024) {
    LFMQ_CHECK_HIP(hipFuncSetAttribute(
        (const void*)attn_latent_decode_mfma<KS, NT, MT>,
        hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds));
    set = true;
  }
  hipLaunchKernelGGL(
      (attn_latent_decode_mfma<KS, NT, MT>),
      dim3(A.splits, (A.heads + MT * 16 - 1) / (MT * 16), sv.b), dim3(TPB),
      lds, stream, sv, A);
  return hipGetLastError();
}

}  // namespace

bool lfmq_attn_latent_decode_mfma_ok(const void* q, const void* ring,
                                     int rank, int rot) {
  return rank % 8 == 0 && rot % 8 == 0 && rank <= 512 && rank + rot <= 576 &&
         (((u64)q | (u64)ring) & 15) == 0;
}

hipError_t lfmq_attn_latent_decode_mfma(const void* q, const void* ring,
                                        const SeqView& sv, void* part,
                                        int heads, int rank, int rot,
                                        int window, int cap, int splits,
                                        float scale, hipStream_t stream) {
  LArgs A{(const bf16_t*)q, (const bf16_t*)ring, (float*)part, heads, rank,
          rot, window, cap, splits, scale};
  const int ks = (rank + rot + 31) / 32;
#define GO(K, N)                                                             \
  do {                                                                       \
    if (heads <= 16) return launch<K, N, 1>(sv, A, stream);                  \
    return launch<K, N, 2>(sv, A, stream);                                   \
  } while (0)
  if (ks <= 4 && rank <= 128) GO(4, 2);
  if (ks <= 10 && rank <= 256) GO(10, 4);
  GO(18, 8);
#undef GO
}
