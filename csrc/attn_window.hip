// Sliding-window attention with a softmax sink over a two-part key, any
// sizes, 16- or 32-bit storage: the general kernels.  attn_window_mfma.hip
// has the matrix-core forms for aligned 16-bit shapes.
//
// Query row r of sequence s at position p sees keys j with
// p - window < j <= p.  A key is {k1 [d1] per head, k2 [d2] shared by all
// heads}, its value [dv] per head; strides of 0 share a part between
// heads, and `group` query heads share a key/value head.  Key rows come
// from a packed step buffer (row = own_row[s] + j - len0) or, with own_row
// null, from a ring cache (slot * cap + j mod cap).
//
// PROMPT: rotates the query's second part, applies the sink, an output
// gate if there is one and a constant gain, writes 16/32-bit rows.  DECODE (absorbed latent form): takes a
// ready query, emits the partial {sum p v, max, sum p} of one key range.
#include "seq_common.h"

namespace {

constexpr int TPB = 256;
constexpr int KT = 256;   // keys per tile

struct WinArgs {
  int heads, d1, d2, rot_dims, dv, window, cap, splits;
  float scale;
  u64 k1_ld, k1_head, k2_ld, v_ld, v_head, ldg;
  int group;
  u64 ldo;
  float gain;
};

template <typename T, bool DECODE>
__global__ __launch_bounds__(TPB) void attn_window_kernel(
    const T* __restrict__ q, const T* __restrict__ k1,
    const T* __restrict__ k2, const T* __restrict__ vv, SeqView sv,
    const i32* __restrict__ own_row, const float* __restrict__ inv_freq,
    const float* __restrict__ sink, const T* __restrict__ g,
    void* __restrict__ outp, WinArgs A) {
  extern __shared__ float sh[];
  const int D = A.d1 + A.d2;
  float* qs = sh;                 // [D]
  float* acc = qs + D;            // [dv]
  float* ps = acc + A.dv;         // [KT]
  __shared__ float red[4];
  const int row = blockIdx.x, h = blockIdx.y, kh = h / A.group;
  const int s = sv.seq[row];
  const int slot = sv.slots[s];
  const int len0 = sv.lens[slot];
  const int pos = len0 + row - sv.cu[s];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const T* qr = q + ((u64)row * A.heads + h) * D;
  for (int j = threadIdx.x; j < D; j += TPB) qs[j] = ldf(qr + j);
  for (int j = threadIdx.x; j < A.dv; j += TPB) acc[j] = 0.f;
  __syncthreads();
  if (!DECODE) {
    const int half = A.rot_dims / 2;
    for (int j = threadIdx.x; j < half; j += TPB) {
      float sn, c;
      sincosf((float)pos * inv_freq[j], &sn, &c);
      const float a = qs[A.d1 + j], b = qs[A.d1 + half + j];
      qs[A.d1 + j] = a * c - b * sn;
      qs[A.d1 + half + j] = b * c + a * sn;
    }
    __syncthreads();
  }
  int lo = pos < A.window ? 0 : pos - A.window + 1, hi = pos + 1;
  if (DECODE) {   // this workgroup's share of the window
    const int per = (hi - lo + A.splits - 1) / A.splits;
    lo += blockIdx.z * per;
    hi = min(hi, lo + per);
  }
  float m = -INFINITY, l = 0.f;
  for (int t0 = lo; t0 < hi; t0 += KT) {
    const int nk = min(KT, hi - t0);
    // scores: one key per wave at a time, lanes across the dimensions
    for (int i = wave; i < nk; i += TPB / 64) {
      const int j = t0 + i;
      const u64 kr = own_row != nullptr ? (u64)(own_row[s] + j - len0)
                                        : (u64)slot * A.cap + j % A.cap;
      const T* a = k1 + kr * A.k1_ld + kh * A.k1_head;
      const T* b = k2 + kr * A.k2_ld;
      float d = 0.f;
      for (int e = lane; e < A.d1; e += 64) d = fmaf(ldf(a + e), qs[e], d);
      for (int e = lane; e < A.d2; e += 64)
        d = fmaf(ldf(b + e), qs[A.d1 + e], d);
      d = wave_reduce_sum(d);
      if (lane == 0) ps[i] = d * A.scale;
    }
    __syncthreads();
    const float sc = threadIdx.x < nk ? ps[threadIdx.x] : -INFINITY;
    float mx = wave_reduce_max(sc);
    if (lane == 0) red[wave] = mx;
    __syncthreads();
    mx = fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3]));
    const float mn = fmaxf(m, mx);
    const float al = expf(m - mn);
    const float p = threadIdx.x < nk ? expf(sc - mn) : 0.f;
    __syncthreads();
    ps[threadIdx.x] = p;
    const float sum = wave_reduce_sum(p);
    if (lane == 0) red[wave] = sum;
    __syncthreads();
    l = l * al + red[0] + red[1] + red[2] + red[3];
    m = mn;
    for (int e = threadIdx.x; e < A.dv; e += TPB) {
      float o = acc[e] * al;
      for (int i = 0; i < nk; ++i) {
        const int j = t0 + i;
        const u64 kr = own_row != nullptr ? (u64)(own_row[s] + j - len0)
                                          : (u64)slot * A.cap + j % A.cap;
        o = fmaf(ps[i], ldf(vv + kr * A.v_ld + kh * A.v_head + e), o);
      }
      acc[e] = o;
    }
    __syncthreads();
  }
  if (DECODE) {
    float* o = (float*)outp +
               (((u64)s * A.splits + blockIdx.z) * A.heads + h) * (A.dv + 2);
    for (int e = threadIdx.x; e < A.dv; e += TPB) o[e] = acc[e];
    if (threadIdx.x == 0) {
      o[A.dv] = m;
      o[A.dv + 1] = l;
    }
    return;
  }
  const float M = fmaxf(m, sink[h]);
  const float w =
      A.gain * expf(m - M) / (l * expf(m - M) + expf(sink[h] - M));
  T* o = (T*)outp + (u64)row * A.ldo + h * A.dv;
  const T* gr = g + (u64)row * A.ldg + h * A.dv;
  for (int e = threadIdx.x; e < A.dv; e += TPB)
    stf(o + e, acc[e] * w * (g != nullptr ? sigmoid_f(ldf(gr + e)) : 1.f));
}

}  // namespace

// keys/values: packed step buffer, k1/v per head
hipError_t lfmq_attn_window_prompt(
    const void* q, const void* k1, long k1_ld, long k1_head, const void* k2,
    long k2_ld, const void* v, long v_ld, long v_head, const SeqView& sv,
    const void* own_row, const void* inv_freq, const void* sink,
    const void* g, long ldg, void* out, int heads, int d1, int d2,
    int rot_dims, int dv, int window, float scale, bool f32,
    hipStream_t stream) {
  WinArgs A{heads, d1, d2, rot_dims, dv, window, 0, 1, scale, (u64)k1_ld,
            (u64)k1_head, (u64)k2_ld, (u64)v_ld, (u64)v_head, (u64)ldg, 1,
            (u64)heads * dv, 1.f};
  const size_t lds = (size_t)(d1 + d2 + dv + KT) * sizeof(float);
  if (lds > 60 * 1024) return hipErrorInvalidValue;
#define GO(T)                                                                \
  hipLaunchKernelGGL((attn_window_kernel<T, false>), dim3(sv.n, heads),      \
                     dim3(TPB), lds, stream, (const T*)q, (const T*)k1,      \
                     (const T*)k2, (const T*)v, sv, (const i32*)own_row,     \
                     (const float*)inv_freq, (const float*)sink,             \
                     (const T*)g, out, A)
  if (f32) GO(float); else GO(bf16_t);
#undef GO
  return hipGetLastError();
}

// latent cache ring [slots, cap, rank + rot]; q [b, heads, rank + rot];
// part [b, splits, heads, rank + 2]
hipError_t lfmq_attn_window_decode(const void* q, const void* ring,
                                   const SeqView& sv, void* part, int heads,
                                   int rank, int rot, int window, int cap,
                                   int splits, float scale, bool f32,
                                   hipStream_t stream) {
  const u64 d = rank + rot;
  WinArgs A{heads, rank, rot, 0, rank, window, cap, splits, scale,
            d, 0, d, d, 0, 0, 1, 0, 1.f};
  const size_t lds = (size_t)(d + rank + KT) * sizeof(float);
  if (lds > 60 * 1024) return hipErrorInvalidValue;
#define GO(T)                                                                \
  hipLaunchKernelGGL((attn_window_kernel<T, true>),                          \
                     dim3(sv.b, heads, splits), dim3(TPB), lds, stream,      \
                     (const T*)q, (const T*)ring, (const T*)ring + rank,     \
                     (const T*)ring, sv, (const i32*)nullptr,                \
                     (const float*)nullptr, (const float*)nullptr,           \
                     (const T*)nullptr, part, A)
  if (f32) GO(float); else GO(bf16_t);
#undef GO
  return hipGetLastError();
}

// grouped queries over a key/value cache: kc [slots, cap, heads / group,
// dim], vc [.., dv]; q [n, heads, dim] ready; out rows of stride ldo.
// Every position from 0 on is seen; any number of tokens per sequence.
hipError_t lfmq_attn_grouped(const void* q, const void* kc, const void* vc,
                             const SeqView& sv, const void* sink, void* out,
                             long ldo, int heads, int group, int dim, int dv,
                             int cap, float scale, float gain, bool f32,
                             hipStream_t stream) {
  const u64 kv = heads / group;
  WinArgs A{heads, dim, 0, 0, dv, INT32_MAX, cap, 1, scale, kv * dim,
            (u64)dim, 0, kv * dv, (u64)dv, 0, group, (u64)ldo, gain};
  const size_t lds = (size_t)(dim + dv + KT) * sizeof(float);
  if (lds > 60 * 1024) return hipErrorInvalidValue;
#define GO(T)                                                                \
  hipLaunchKernelGGL((attn_window_kernel<T, false>), dim3(sv.n, heads),      \
                     dim3(TPB), lds, stream, (const T*)q, (const T*)kc,      \
                     (const T*)kc, (const T*)vc, sv, (const i32*)nullptr,    \
                     (const float*)nullptr, (const float*)sink,              \
                     (const T*)nullptr, out, A)
  if (f32) GO(float); else GO(bf16_t);
#undef GO
  return hipGetLastError();
}
