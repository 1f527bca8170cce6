// Decode attention of grouped queries over the key/value cache (one token
// per sequence, 16-bit, aligned sizes; attn_window.hip: lfmq_attn_grouped
// states the semantics and covers every other shape).
//
// A workgroup = one key range x up to GH query heads of one key/value head,
// 4 waves.  A wave takes 32 keys at a time on its own, no barriers: scores
// on the matrix cores with the keys as rows (a lane reads 16 bytes of a
// key straight from the cache), the online softmax per head across the
// lanes, weights through a small LDS slab, and the weighted sum in fp32 on
// the vector units (a lane owns 8 value columns, so values need no
// transposition; at these head counts the cache read is the bound).  The
// waves' results meet once at the end.  With more than one key range the
// partial {sum p v, max, sum p} goes to the merge kernel, which lets the
// sink into the denominator; otherwise the workgroup finishes itself.
#include "seq_common.h"

namespace {

constexpr int TPB = 256, NW = 4, KT = 32;

struct GArgs {
  const bf16_t *q, *kc, *vc;
  const float* sink;
  float* part;
  bf16_t* out;
  u64 ldo;
  int heads, group, dim, dv, cap, splits;
  float scale, gain;
};

template <int KS, int LPR, int GH>
__global__ __launch_bounds__(TPB) void attn_grouped_decode_kernel(SeqView sv,
                                                                  GArgs A) {
  constexpr int RPP = 64 / LPR;          // value rows a pass
  constexpr int NP = KT / RPP;           // passes a tile
  constexpr int DV = LPR * 8;
  __shared__ __attribute__((aligned(16))) float ps[NW][KT][GH];
  __shared__ __attribute__((aligned(16))) float al_s[NW][GH];
  __shared__ float ml[NW][GH][2];
  __shared__ float ws[NW][GH][DV + 1];
  const int s = blockIdx.z;
  const int htiles = (A.group + GH - 1) / GH;
  const int kh = blockIdx.y / htiles, ht = blockIdx.y % htiles;
  const int h0 = kh * A.group + ht * GH;           // first query head
  const int nh = min(GH, A.group - ht * GH);
  const int slot = sv.slots[s];
  const int len = min(sv.lens[slot] + 1, A.cap);
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  const int l15 = lane & 15, l4 = lane >> 4;
  const int per =
      ((len + A.splits - 1) / A.splits + KT - 1) / KT * KT;
  const int lo = min(len, (int)blockIdx.x * per), hi = min(len, lo + per);
  const u64 kv = A.heads / A.group;
  const bf16_t* K = A.kc + ((u64)slot * A.cap * kv + kh) * A.dim;
  const bf16_t* V = A.vc + ((u64)slot * A.cap * kv + kh) * A.dv;
  const u64 ldk = kv * A.dim, ldv_ = kv * A.dv;
  const s16x8 z8 = {0, 0, 0, 0, 0, 0, 0, 0};

  s16x8 qf[KS];
  {
    const bf16_t* qr = A.q + ((u64)s * A.heads + h0 + l15) * A.dim;
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
      const int k = ks * 32 + l4 * 8;
      qf[ks] = (l15 < nh && k < A.dim) ? *(const s16x8*)(qr + k) : z8;
    }
  }
  float m = -INFINITY, l = 0.f;          // of head l15
  float acc[GH][8] = {};
  const int vrow = lane / LPR, vcol = (lane % LPR) * 8;
  const bool vok = vcol < A.dv;

  for (int t0 = lo + wave * KT; t0 < hi; t0 += NW * KT) {
    s16x8 kf[2][KS];
    u32x4 vv[NP];
#pragma unroll
    for (int mt = 0; mt < 2; ++mt) {
      const bf16_t* kr = K + (u64)min(t0 + mt * 16 + l15, hi - 1) * ldk;
#pragma unroll
      for (int ks = 0; ks < KS; ++ks) {
        const int k = ks * 32 + l4 * 8;
        kf[mt][ks] = k < A.dim ? *(const s16x8*)(kr + k) : z8;
      }
    }
#pragma unroll
    for (int i = 0; i < NP; ++i) {
      const u32x4 z = {0, 0, 0, 0};
      vv[i] = vok ? *(const u32x4*)(V + (u64)min(t0 + i * RPP + vrow, hi - 1) *
                                            ldv_ + vcol)
                  : z;
    }
    f32x4 sc[2] = {};
#pragma unroll
    for (int ks = 0; ks < KS; ++ks)
#pragma unroll
      for (int mt = 0; mt < 2; ++mt)
        sc[mt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[mt][ks], qf[ks],
                                                         sc[mt], 0, 0, 0);
    float mx = -INFINITY;
#pragma unroll
    for (int mt = 0; mt < 2; ++mt)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const bool ok = t0 + mt * 16 + l4 * 4 + r < hi;
        sc[mt][r] = ok ? sc[mt][r] * A.scale : -INFINITY;
        mx = fmaxf(mx, sc[mt][r]);
      }
    mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
    mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
    const float mn = fmaxf(m, mx);             // a tile has a visible key
    const float al = __expf(m - mn);
    float sum = 0.f;
#pragma unroll
    for (int mt = 0; mt < 2; ++mt)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const float p = __expf(sc[mt][r] - mn);
        sum += p;
        if (l15 < GH) ps[wave][mt * 16 + l4 * 4 + r][l15] = p;
      }
    sum += __shfl_xor(sum, 16, 64);
    sum += __shfl_xor(sum, 32, 64);
    l = l * al + sum;
    m = mn;
    if (lane < GH) al_s[wave][lane] = al;
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
#pragma unroll
    for (int h = 0; h < GH; ++h) {
      const float a = al_s[wave][h];
#pragma unroll
      for (int e = 0; e < 8; ++e) acc[h][e] *= a;
    }
#pragma unroll
    for (int i = 0; i < NP; ++i) {
      float v[8];
#pragma unroll
      for (int e = 0; e < 4; ++e) bf16x2_to_f32(vv[i][e], v[2 * e], v[2 * e + 1]);
      const float* pr = ps[wave][i * RPP + vrow];
#pragma unroll
      for (int h = 0; h < GH; ++h) {
        const float p = pr[h];
#pragma unroll
        for (int e = 0; e < 8; ++e) acc[h][e] = fmaf(p, v[e], acc[h][e]);
      }
    }
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");  // ps is read
  }

  // rows of one wave, then the waves
#pragma unroll
  for (int h = 0; h < GH; ++h)
#pragma unroll
    for (int e = 0; e < 8; ++e) {
#pragma unroll
      for (int o = LPR; o < 64; o <<= 1)
        acc[h][e] += __shfl_xor(acc[h][e], o, 64);
      if (lane < LPR) ws[wave][h][vcol + e] = acc[h][e];
    }
  if (lane < GH) {
    ml[wave][lane][0] = m;
    ml[wave][lane][1] = l;
  }
  __syncthreads();
  for (int id = tid; id < nh * A.dv; id += TPB) {
    const int h = id / A.dv, e = id % A.dv;
    float M = fmaxf(fmaxf(ml[0][h][0], ml[1][h][0]),
                    fmaxf(ml[2][h][0], ml[3][h][0]));
    const bool last = A.splits == 1;
    if (last) M = fmaxf(M, A.sink[h0 + h]);
    float o = 0.f, L = 0.f;
    if (M > -INFINITY) {
#pragma unroll
      for (int w = 0; w < NW; ++w) {
        const float c = __expf(ml[w][h][0] - M);
        o = fmaf(c, ws[w][h][e], o);
        L = fmaf(c, ml[w][h][1], L);
      }
    }
    if (last) {
      L += __expf(A.sink[h0 + h] - M);
      stf(A.out + (u64)s * A.ldo + (u64)(h0 + h) * A.dv + e, o * A.gain / L);
      continue;
    }
    float* p = A.part + (((u64)s * A.splits + blockIdx.x) * A.heads + h0 + h) *
                            (A.dv + 2);
    p[e] = o;
    if (e == 0) {
      p[A.dv] = M;
      p[A.dv + 1] = L;
    }
  }
}

// part [b, splits, heads, dv + 2]
__global__ __launch_bounds__(256) void attn_merge_kernel(
    const float* __restrict__ part, const float* __restrict__ sink,
    bf16_t* __restrict__ out, u64 ldo, int heads, int dv, int splits,
    float gain) {
  __shared__ float wt[64];
  const int h = blockIdx.x, s = blockIdx.y;
  const u64 sp = (u64)heads * (dv + 2);
  const float* p = part + ((u64)s * splits * heads + h) * (dv + 2);
  if (threadIdx.x < 64) {
    const int c = threadIdx.x;
    const bool on = c < splits;
    const float mc = on ? p[c * sp + dv] : -INFINITY;
    const float M = fmaxf(wave_reduce_max(mc), sink[h]);
    const float e = on ? __expf(mc - M) : 0.f;
    const float L =
        wave_reduce_sum(on ? e * p[c * sp + dv + 1] : 0.f) + __expf(sink[h] - M);
    wt[c] = e * gain / L;
  }
  __syncthreads();
  for (int e = threadIdx.x; e < dv; e += blockDim.x) {
    float a = 0.f;
#pragma unroll 8
    for (int c = 0; c < splits; ++c) a = fmaf(wt[c], p[c * sp + e], a);
    stf(out + (u64)s * ldo + (u64)h * dv + e, a);
  }
}

template <int KS, int LPR>
hipError_t launch(const SeqView& sv, const GArgs& A, hipStream_t stream) {
  const int gh = A.group <= 4 ? 4 : 8;
  const dim3 grid(A.splits, A.heads / A.group * ((A.group + gh - 1) / gh),
                  sv.b);
  if (gh == 4)
    hipLaunchKernelGGL((attn_grouped_decode_kernel<KS, LPR, 4>), grid,
                       dim3(TPB), 0, stream, sv, A);
  else
    hipLaunchKernelGGL((attn_grouped_decode_kernel<KS, LPR, 8>), grid,
                       dim3(TPB), 0, stream, sv, A);
  return hipGetLastError();
}

}  // namespace

// one key range per workgroup: enough of them to fill the chip, none
// shorter than a tile of every wave, at most 64 (a wave merges them)
int lfmq_attn_grouped_splits(int b, int heads, int group, int cap) {
  const int gh = group <= 4 ? 4 : 8;
  const int wgs = b * (heads / group) * ((group + gh - 1) / gh);
  int n = (1024 + wgs - 1) / wgs;
  const int most = (cap + NW * KT - 1) / (NW * KT);
  n = n < most ? n : most;
  return n < 1 ? 1 : (n > 64 ? 64 : n);
}

// part: splits > 1 only, [b, splits, heads, dv + 2] fp32
hipError_t lfmq_attn_grouped_decode(const void* q, const void* kc,
                                    const void* vc, const SeqView& sv,
                                    const void* sink, void* part, void* out,
                                    long ldo, int heads, int group, int dim,
                                    int dv, int cap, int splits, float scale,
                                    float gain, hipStream_t stream) {
  GArgs A{(const bf16_t*)q, (const bf16_t*)kc, (const bf16_t*)vc,
          (const float*)sink, (float*)part, (bf16_t*)out, (u64)ldo, heads,
          group, dim, dv, cap, splits, scale, gain};
  hipError_t e;
#define GO(K)                                                                \
  do {                                                                       \
    if (dv <= 64) e = launch<K, 8>(sv, A, stream);                           \
    else if (dv <= 128) e = launch<K, 16>(sv, A, stream);                    \
    else e = launch<K, 32>(sv, A, stream);                                   \
  } while (0)
  if (dim <= 64) GO(2);
  else if (dim <= 128) GO(4);
  else GO(8);
#undef GO
  if (e != hipSuccess || splits == 1) return e;
  hipLaunchKernelGGL(attn_merge_kernel, dim3(heads, sv.b),
                     dim3(dv <= 64 ? 64 : (dv <= 128 ? 128 : 256)), 0, stream,
                     (const float*)part, (const float*)sink, (bf16_t*)out,
                     (u64)ldo, heads, dv, splits, gain);
  return hipGetLastError();
}
