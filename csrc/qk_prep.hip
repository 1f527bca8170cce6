// Grouped-query attention ahead of its score kernels: one pass over the
// projection's [ q | k | v ] columns norms all query rows and all key rows
// of a token (each over the whole projection), rotates both, and writes the
// queries to a buffer and keys and values into the cache, where position p
// of slot s is row s * cap + p.
//
// One workgroup a token: the normed rows meet in LDS, since a rotation
// pairs dimension i of a head with i + half.  The angles' sines and cosines
// are computed once for all heads.
#include "seq_common.h"

namespace {

template <typename T, int VEC, int TPB>
__global__ __launch_bounds__(TPB) void qk_prep_kernel(
    const T* __restrict__ in, u64 ld, SeqView sv,
    const float* __restrict__ wq, const float* __restrict__ wk,
    const float* __restrict__ inv_freq, T* __restrict__ q,
    T* __restrict__ kc, T* __restrict__ vc, int cap, int nq, int nk, int nv,
    int dim, int half, float eps) {
  extern __shared__ float sh[];
  float* buf = sh;                 // [nq + nk]
  float* cs = buf + nq + nk;       // [half]
  float* sn = cs + half;           // [half]
  __shared__ float red[2][TPB / 64];
  const int row = blockIdx.x;
  const int s = sv.seq[row], slot = sv.slots[s];
  const int pos = sv.lens[slot] + row - sv.cu[s];
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const T* src = in + (u64)row * ld;
  float sq = 0.f, sk = 0.f;
  for (int j = threadIdx.x * VEC; j < nq + nk; j += TPB * VEC) {
    float a[VEC], ss = 0.f;
    ldv<T, VEC>(src + j, a);
#pragma unroll
    for (int e = 0; e < VEC; ++e) ss = fmaf(a[e], a[e], ss);
    if (j < nq) sq += ss; else sk += ss;
    stv<float, VEC>(buf + j, a);
  }
  for (int j = threadIdx.x; j < half; j += TPB)
    sincosf((float)pos * inv_freq[j], sn + j, cs + j);
  sq = wave_reduce_sum(sq);
  sk = wave_reduce_sum(sk);
  if (lane == 0) {
    red[0][wave] = sq;
    red[1][wave] = sk;
  }
  __syncthreads();
  sq = sk = 0.f;
#pragma unroll
  for (int i = 0; i < TPB / 64; ++i) {
    sq += red[0][i];
    sk += red[1][i];
  }
  const float iq = 1.f / sqrtf(sq / (float)nq + eps);
  const float ik = 1.f / sqrtf(sk / (float)nk + eps);
  T* qo = q + (u64)row * nq;
  const bool fits = pos < cap;
  T* ko = kc + ((u64)slot * cap + pos) * nk;
  T* vo = vc + ((u64)slot * cap + pos) * nv;
  for (int j = threadIdx.x * VEC; j < nq + nk; j += TPB * VEC) {
    const bool isq = j < nq;
    const int c = isq ? j : j - nq, d = c % dim;
    const float inv = isq ? iq : ik;
    const float* w = isq ? wq : wk;
    float a[VEC], g[VEC];
    ldv<float, VEC>(buf + j, a);
    ldv<float, VEC>(w + c, g);
#pragma unroll
    for (int e = 0; e < VEC; ++e) a[e] = a[e] * inv * g[e];
    if (d < 2 * half) {
      const int o = d < half ? half : -half, t = d < half ? d : d - half;
      const float sgn = d < half ? -1.f : 1.f;
      float b[VEC];
      ldv<float, VEC>(buf + j + o, b);
      ldv<float, VEC>(w + c + o, g);
#pragma unroll
      for (int e = 0; e < VEC; ++e)
        a[e] = a[e] * cs[t + e] + sgn * (b[e] * inv * g[e]) * sn[t + e];
    }
    if (isq) stv<T, VEC>(qo + c, a);
    else if (fits) stv<T, VEC>(ko + c, a);
  }
  if (!fits) return;
  const T* vs = src + nq + nk;
  for (int j = threadIdx.x * VEC; j < nv; j += TPB * VEC) {
    float a[VEC];
    ldv<T, VEC>(vs + j, a);
    stv<T, VEC>(vo + j, a);
  }
}

}  // namespace

hipError_t lfmq_qk_prep(const void* in, long ld, const SeqView& sv,
                        const void* wq, const void* wk, const void* inv_freq,
                        void* q, void* kc, void* vc, int cap, int nq, int nk,
                        int nv, int dim, int half, float eps, bool f32,
                        hipStream_t stream) {
  const size_t lds = ((size_t)nq + nk + 2 * half) * sizeof(float);
  if (lds > 64 * 1024) return hipErrorInvalidValue;
  const bool v4 = ((ld | dim | half | nv) & 3) == 0 &&
                  (((u64)in | (u64)wq | (u64)wk | (u64)q | (u64)kc |
                    (u64)vc) & 15) == 0;
  // few rows: more threads each
#define GO(T, V)                                                             \
  do { if (sv.n < 512) GOT(T, V, 1024); else GOT(T, V, 256); } while (0)
#define GOT(T, V, N)                                                         \
  hipLaunchKernelGGL((qk_prep_kernel<T, V, N>), dim3(sv.n), dim3(N), lds,    \
                     stream, (const T*)in, (u64)ld, sv, (const float*)wq,    \
                     (const float*)wk, (const float*)inv_freq, (T*)q,        \
                     (T*)kc, (T*)vc, cap, nq, nk, nv, dim, half, eps)
  if (f32) { if (v4) GO(float, 4); else GO(float, 1); }
  else { if (v4) GO(bf16_t, 4); else GO(bf16_t, 1); }
#undef GOT
#undef GO
  return hipGetLastError();
}
