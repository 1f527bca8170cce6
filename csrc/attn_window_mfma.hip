// Matrix-core form of the windowed sink attention for 16-bit prompts
// (attn_window.hip states the semantics and covers every other shape).
//
// One workgroup = 4 waves x QT * 16 queries of one head, key tiles of 64
// from the window's first key on.  Scores are computed transposed (keys as
// rows, queries as columns), so that a lane holds 16 keys of one query: the
// softmax needs two shuffles a tile, and the weights are already the right
// operand of the product with the values, transposed as well (the order of
// the keys inside a step is the accumulator's, on both sides).  Both key
// parts are staged side by side in LDS (16 B row pad), values transposed
// (Vt[d][key], XOR swizzled in 16-byte blocks so that the packed two-key
// writes and the fragment reads both spread over the banks).  The next tile
// is in flight while this one is multiplied.  Queries are staged and rotated
// once.  Scores and the online softmax stay in fp32 registers; the sink
// starts the running maximum and denominator, so a row is never empty.  The
// epilogue applies 1/l and the output gate.
#include "seq_common.h"

namespace {

constexpr int TPB = 256;
constexpr int BN = 64;

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
  bool v4;               // four columns of g and out may be moved at once
};

__device__ __forceinline__ u32 swz(u32 row) { return (row ^ (row >> 3)) & 7; }

__device__ __forceinline__ u32 pack2(float a, float b) {
  const bf16x2_native v = {(__bf16)a, (__bf16)b};
  return __builtin_bit_cast(u32, v);
}

template <int KS, int VT, int QT>
__global__ __launch_bounds__(TPB, 2) void attn_window_prompt_mfma(SeqView sv,
                                                                  PArgs A) {
  constexpr int QKP = KS * 32, VP = VT * 16, BM = 64 * QT;
  constexpr int KROW = QKP * 2 + 16;
  constexpr int NK = BN * (QKP / 8) / TPB;             // staging items
  constexpr int NV = (BN / 2) * (VP / 8) / TPB;
  extern __shared__ __attribute__((aligned(16))) char smem[];
  char* ldsK = smem;
  char* ldsV = ldsK + BN * KROW;
  // the last queries see the most keys: they start first
  const int q0 = (gridDim.x - 1 - blockIdx.x) * BM;
  const int s = blockIdx.z, h = blockIdx.y, kh = h / A.group;
  const int row0 = sv.cu[s], cnt = sv.cu[s + 1] - row0;
  if (q0 >= cnt) return;
  const int slot = sv.slots[s], len0 = sv.lens[slot];
  const int tid = threadIdx.x, lane = tid & 63;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int l15 = lane & 15, l4 = lane >> 4;
  const int D = A.d1 + A.d2;
  const int half = A.rot_dims / 2;

  // ---- queries, 64 at a time: stage, rotate the second part, keep ----
  s16x8 qf[QT][KS];
#pragma unroll
  for (int qt = 0; qt < QT; ++qt) {
    // this pass: query tile qt of every wave
    __syncthreads();
    for (int c = tid; c < 64 * (QKP / 8); c += TPB) {
      const int r = c / (QKP / 8), e0 = (c % (QKP / 8)) * 8;
      const int qr = q0 + (r >> 4) * (16 * QT) + qt * 16 + (r & 15);
      u32x4 d = {0, 0, 0, 0};
      if (qr < cnt && e0 < D)
        d = *(const u32x4*)(A.q + ((u64)(row0 + qr) * A.heads + h) * D + e0);
      *(u32x4*)(ldsK + r * KROW + e0 * 2) = d;
    }
    __syncthreads();
    for (int c = tid; c < 64 * half; c += TPB) {
      const int r = c / half, j = c % half;
      const int qr = q0 + (r >> 4) * (16 * QT) + qt * 16 + (r & 15);
      unsigned short* p = (unsigned short*)(ldsK + r * KROW) + A.d1 + j;
      float sn, cs;
      sincosf((float)(len0 + qr) * A.inv_freq[j], &sn, &cs);
      const float u = bf16_bits_to_f32(p[0]), w = bf16_bits_to_f32(p[half]);
      p[0] = (unsigned short)f32_to_bf16_bits_rne(u * cs - w * sn);
      p[half] = (unsigned short)f32_to_bf16_bits_rne(w * cs + u * sn);
    }
    __syncthreads();
#pragma unroll
    for (int ks = 0; ks < KS; ++ks)
      qf[qt][ks] = *(const s16x8*)(ldsK + (wave * 16 + l15) * KROW +
                                   (ks * 32 + l4 * 8) * 2);
  }

  // softmax in powers of two
  constexpr float LOG2E = 1.4426950408889634f;
  const float sc2 = A.scale * LOG2E, snk = A.sink[h] * LOG2E;
  float m[QT], l[QT];
#pragma unroll
  for (int qt = 0; qt < QT; ++qt) {
    m[qt] = snk;
    l[qt] = 1.f;
  }
  f32x4 oacc[QT][VT] = {};

  const int p_lo = len0 + q0, p_hi = len0 + min(q0 + BM, cnt) - 1;
  const int lo = p_lo < A.window ? 0 : p_lo - A.window + 1, hi = p_hi + 1;
  // row of key 0: in the step's key buffer, or in the cache
  const long base = A.own_row != nullptr ? (long)A.own_row[s] - len0
                                         : (long)slot * A.cap;
  const int w_lo = p_lo + wave * (16 * QT), w_hi = w_lo + 16 * QT - 1;

  u32x4 xk[NK], xa[NV], xb[NV];
  auto fetch = [&](int t0) {
    const u32x4 z = {0, 0, 0, 0};
#pragma unroll
    for (int i = 0; i < NK; ++i) {
      const int c = i * TPB + tid;
      const int key = c / (QKP / 8), e0 = (c % (QKP / 8)) * 8;
      const u64 kr = (u64)(base + min(t0 + key, hi - 1));
      xk[i] = z;
      if (e0 < A.d1)
        xk[i] = *(const u32x4*)(A.k1 + kr * A.k1_ld + kh * A.d1 + e0);
      else if (e0 < D)
        xk[i] = *(const u32x4*)(A.k2 + kr * A.k2_ld + (e0 - A.d1));
    }
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int c = i * TPB + tid;
      const int kp = c / (VP / 8), dg = c % (VP / 8);
      xa[i] = z;
      xb[i] = z;
      if (dg * 8 < A.dv) {
        const u64 ra = (u64)(base + min(t0 + 2 * kp, hi - 1));
        const u64 rb = (u64)(base + min(t0 + 2 * kp + 1, hi - 1));
        xa[i] = *(const u32x4*)(A.v + ra * A.v_ld + kh * A.dv + dg * 8);
        xb[i] = *(const u32x4*)(A.v + rb * A.v_ld + kh * A.dv + dg * 8);
      }
    }
  };
  fetch(lo);
  for (int t0 = lo; t0 < hi; t0 += BN) {
    __syncthreads();                 // the last tile is consumed
#pragma unroll
    for (int i = 0; i < NK; ++i) {
      const int c = i * TPB + tid;
      *(u32x4*)(ldsK + c / (QKP / 8) * KROW + (c % (QKP / 8)) * 16) = xk[i];
    }
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int c = i * TPB + tid;
      const int kp = c / (VP / 8), dg = c % (VP / 8);
      const u32 blk = kp >> 2, off = (kp & 3) * 4;
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        const u32 d = dg * 8 + e;
        // the same 16 bits of both keys
        const u32 v = __builtin_amdgcn_perm(xb[i][e >> 1], xa[i][e >> 1],
                                            e & 1 ? 0x07060302u : 0x05040100u);
        *(u32*)(ldsV + d * 128 + ((blk ^ swz(d)) << 4) + off) = v;
      }
    }
    if (t0 + BN < hi) fetch(t0 + BN);
    __syncthreads();
    if (t0 > w_hi || w_lo - (t0 + BN - 1) >= A.window) continue;  // none seen

    f32x4 sc[QT][BN / 16] = {};
#pragma unroll
    for (int ks = 0; ks < KS; ++ks)
#pragma unroll
      for (int nt = 0; nt < BN / 16; ++nt) {
        const s16x8 kf = *(const s16x8*)(ldsK + (nt * 16 + l15) * KROW +
                                         (ks * 32 + l4 * 8) * 2);
#pragma unroll
        for (int qt = 0; qt < QT; ++qt)
          sc[qt][nt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
              kf, qf[qt][ks], sc[qt][nt], 0, 0, 0);
      }
    // a tile that every query of this wave sees whole needs no mask
    const bool whole = t0 + BN - 1 <= w_lo && w_hi - t0 < A.window &&
                       t0 + BN <= hi;
    s16x8 pf[QT][BN / 32];
#pragma unroll
    for (int qt = 0; qt < QT; ++qt) {
      if (!whole) {
        const int pos = w_lo + qt * 16 + l15;
#pragma unroll
        for (int nt = 0; nt < BN / 16; ++nt)
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            const int j = t0 + nt * 16 + l4 * 4 + r;
            const bool ok = j <= pos && pos - j < A.window && j < hi;
            sc[qt][nt][r] = ok ? sc[qt][nt][r] * sc2 : -INFINITY;
          }
      } else {
#pragma unroll
        for (int nt = 0; nt < BN / 16; ++nt) sc[qt][nt] *= sc2;
      }
      float mx = m[qt];
#pragma unroll
      for (int nt = 0; nt < BN / 16; ++nt)
#pragma unroll
        for (int r = 0; r < 4; ++r) mx = fmaxf(mx, sc[qt][nt][r]);
      mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
      mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
      if (__any(mx > m[qt])) {
        const float al = __builtin_amdgcn_exp2f(m[qt] - mx);
        m[qt] = mx;
        l[qt] *= al;
#pragma unroll
        for (int on = 0; on < VT; ++on) oacc[qt][on] *= al;
      }
      float ps = 0.f;
#pragma unroll
      for (int nt = 0; nt < BN / 16; ++nt)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          sc[qt][nt][r] = __builtin_amdgcn_exp2f(sc[qt][nt][r] - m[qt]);
          ps += sc[qt][nt][r];
        }
      ps += __shfl_xor(ps, 16, 64);
      ps += __shfl_xor(ps, 32, 64);
      l[qt] += ps;
#pragma unroll
      for (int k2 = 0; k2 < BN / 32; ++k2) {
        const f32x4 a = sc[qt][2 * k2], b = sc[qt][2 * k2 + 1];
        const u32x4 v = {pack2(a[0], a[1]), pack2(a[2], a[3]),
                         pack2(b[0], b[1]), pack2(b[2], b[3])};
        pf[qt][k2] = __builtin_bit_cast(s16x8, v);
      }
    }
    // keys of a step, in the scores' order: 16 (2 k2) + 4 l4 + 0..3, then
    // the same of the next 16
#pragma unroll
    for (int k2 = 0; k2 < BN / 32; ++k2)
#pragma unroll
      for (int on = 0; on < VT; ++on) {
        const u32 d = on * 16 + l15, blk = k2 * 4 + (l4 >> 1);
        const char* vr = ldsV + d * 128 + (l4 & 1) * 8;
        const u32x2 a = *(const u32x2*)(vr + ((blk ^ swz(d)) << 4));
        const u32x2 b = *(const u32x2*)(vr + (((blk + 2) ^ swz(d)) << 4));
        const u32x4 v = {a[0], a[1], b[0], b[1]};
        const s16x8 vf = __builtin_bit_cast(s16x8, v);
#pragma unroll
        for (int qt = 0; qt < QT; ++qt)
          oacc[qt][on] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
              vf, pf[qt][k2], oacc[qt][on], 0, 0, 0);
      }
  }

  // a lane holds four consecutive columns of one query
#pragma unroll
  for (int qt = 0; qt < QT; ++qt) {
    const int qr = q0 + wave * (16 * QT) + qt * 16 + l15;
    if (qr >= cnt) continue;
    const float inv = A.gain / l[qt];
    const u64 row = row0 + qr;
    const bf16_t* gr = A.g + row * A.ldg + h * A.dv;
    bf16_t* o = A.out + row * A.ldo + h * A.dv;
#pragma unroll
    for (int on = 0; on < VT; ++on) {
      const int e = on * 16 + l4 * 4;
      if (e >= A.dv) continue;
      float y[4], g[4];
#pragma unroll
      for (int r = 0; r < 4; ++r) y[r] = oacc[qt][on][r] * inv;
      if (A.g != nullptr) {
        if (A.v4) {
          ldf4(gr + e, g);
        } else {
#pragma unroll
          for (int r = 0; r < 4; ++r) g[r] = ldf(gr + e + r);
        }
#pragma unroll
        for (int r = 0; r < 4; ++r) y[r] *= sigmoid_f(g[r]);
      }
      if (A.v4) {
        stf4(o + e, y);
      } else {
#pragma unroll
        for (int r = 0; r < 4; ++r) stf(o + e + r, y[r]);
      }
    }
  }
}

template <int KS, int VT>
hipError_t launch(const SeqView& sv, const PArgs& A, int max_count,
                  hipStream_t stream) {
  // two query tiles a wave where their accumulators fit the registers
  constexpr int QT = KS <= 4 && VT <= 8 ? 2 : 1;
  constexpr size_t lds = (size_t)BN * (KS * 64 + 16) + VT * 16 * 128;
  static_assert(lds <= 80 * 1024, "two workgroups share a CU");
  static bool set = false;
  if (!set && lds > 64 * 1024) {
    LFMQ_CHECK_HIP(hipFuncSetAttribute(
        (const void*)attn_window_prompt_mfma<KS, VT, QT>,
        hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds));
    set = true;
  }
  hipLaunchKernelGGL((attn_window_prompt_mfma<KS, VT, QT>),
                     dim3((max_count + 64 * QT - 1) / (64 * QT), A.heads, sv.b),
                     dim3(TPB), lds, stream, sv, A);
  return hipGetLastError();
}

bool al8(const void* p) { return ((u64)p & 7) == 0; }

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
          window, scale, 1, 0, (u64)heads * dv, 1.f,
          ldg % 4 == 0 && al8(g) && al8(out)};
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
          INT32_MAX, scale, group, cap, (u64)ldo, gain,
          ldo % 4 == 0 && al8(out)};
  return dispatch(sv, A, max_count, stream);
}
