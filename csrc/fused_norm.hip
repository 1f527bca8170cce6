// Norms around the fp32 residual stream.
//
// add_norm: x += y (the previous sublayer's output, 16-bit or fp32) and
// h = x * rsqrt(mean(x^2) + eps) * (bias + w) in one pass over the row,
// with an optional SIDE PROJECTION p = h * Wp^T + bp of a few outputs in
// fp32 (the gates of a recurrent layer must not round to 16 bits, and the
// row is in LDS already).  bias 1 is for weights kept as offsets from one,
// bias 0 for plain ones.
//
// One wave owns a row; a workgroup takes `rpw` rows, so that the side
// projection's weights are read once for all of them.  With one row per
// workgroup (decode) all waves share the row instead.
//
// head_norm_gate: o / rms(o) per head, times a weight, times sigmoid(gate).
#include "seq_common.h"

namespace {

template <typename T, int VEC, bool SHARED>
__global__ __launch_bounds__(512) void add_norm_kernel(
    float* __restrict__ x, const T* __restrict__ y,
    const float* __restrict__ w, float bias, T* __restrict__ h, int n,
    int width, float eps, const T* __restrict__ wp,
    const float* __restrict__ bp, float* __restrict__ p, int np) {
  extern __shared__ float rows[];  // [rows per workgroup][width]
  __shared__ float red[8];
  const int wave = threadIdx.x / LFMQ_WAVE, lane = threadIdx.x % LFMQ_WAVE;
  const int nwave = blockDim.x / LFMQ_WAVE;
  constexpr int rpw = SHARED ? 1 : 4;
  const int row0 = blockIdx.x * rpw;
  const int lr = SHARED ? 0 : wave;           // local row of this thread
  const int row = row0 + lr;
  const int t0 = SHARED ? threadIdx.x : lane;
  const int step = SHARED ? blockDim.x : LFMQ_WAVE;
  const bool live = row < n;
  float* hr = rows + (u64)lr * width;
  float ss = 0.f;
  if (live) {
    float* xr = x + (u64)row * width;
    for (int j = t0 * VEC; j < width; j += step * VEC) {
      float a[VEC];
      ldv<float, VEC>(xr + j, a);
      if (y != nullptr) {
        float c[VEC];
        ldv<T, VEC>(y + (u64)row * width + j, c);
#pragma unroll
        for (int e = 0; e < VEC; ++e) a[e] += c[e];
        stv<float, VEC>(xr + j, a);
      }
#pragma unroll
      for (int e = 0; e < VEC; ++e) ss = fmaf(a[e], a[e], ss);
      stv<float, VEC>(hr + j, a);
    }
  }
  ss = wave_reduce_sum(ss);
  if constexpr (SHARED) {
    if (lane == 0) red[wave] = ss;
    __syncthreads();
    ss = 0.f;
    for (int i = 0; i < nwave; ++i) ss += red[i];
  }
  const float inv = 1.f / sqrtf(ss / (float)width + eps);
  if (live) {
    // every thread scales the very elements that it stored
    for (int j = t0 * VEC; j < width; j += step * VEC) {
      float a[VEC], g[VEC];
      ldv<float, VEC>(hr + j, a);
      ldv<float, VEC>(w + j, g);
#pragma unroll
      for (int e = 0; e < VEC; ++e) a[e] = a[e] * inv * (bias + g[e]);
      stv<T, VEC>(h + (u64)row * width + j, a);
      if (wp != nullptr) stv<float, VEC>(hr + j, a);
    }
  }
  if (wp == nullptr) return;
  __syncthreads();
  // wave-strided outputs; each weight row serves all rows of the group
  for (int o = wave; o < np; o += nwave) {
    float acc[rpw];
#pragma unroll
    for (int r = 0; r < rpw; ++r) acc[r] = 0.f;
    for (int j = lane * VEC; j < width; j += LFMQ_WAVE * VEC) {
      float g[VEC];
      ldv<T, VEC>(wp + (u64)o * width + j, g);
#pragma unroll
      for (int r = 0; r < rpw; ++r) {
        float a[VEC];
        ldv<float, VEC>(rows + (u64)r * width + j, a);
#pragma unroll
        for (int e = 0; e < VEC; ++e) acc[r] = fmaf(a[e], g[e], acc[r]);
      }
    }
#pragma unroll
    for (int r = 0; r < rpw; ++r) {
      const float v = wave_reduce_sum(acc[r]);
      if (lane == 0 && row0 + r < n)
        p[(u64)(row0 + r) * np + o] = v + bp[o];
    }
  }
}

template <typename T, int VEC>
__global__ __launch_bounds__(256) void head_norm_gate_kernel(
    const float* __restrict__ o, const T* __restrict__ g, u64 ldg,
    const float* __restrict__ w, T* __restrict__ out, u64 pairs, int heads,
    int v, float eps) {
  const u64 id = (u64)blockIdx.x * (256 / LFMQ_WAVE) + threadIdx.x / LFMQ_WAVE;
  const int lane = threadIdx.x % LFMQ_WAVE;
  if (id >= pairs) return;
  const u64 row = id / heads;
  const int h = id % heads;
  const float* src = o + id * v;
  const T* gr = g + row * ldg + h * v;
  T* dst = out + id * v;
  float ss = 0.f;
#pragma unroll 2
  for (int j = lane * VEC; j < v; j += LFMQ_WAVE * VEC) {
    float a[VEC];
    ldv<float, VEC>(src + j, a);
#pragma unroll
    for (int e = 0; e < VEC; ++e) ss = fmaf(a[e], a[e], ss);
  }
  ss = wave_reduce_sum(ss);
  const float inv = 1.f / sqrtf(ss / (float)v + eps);
#pragma unroll 2
  for (int j = lane * VEC; j < v; j += LFMQ_WAVE * VEC) {
    float a[VEC], c[VEC], k[VEC];
    ldv<float, VEC>(src + j, a);
    ldv<T, VEC>(gr + j, c);
    ldv<float, VEC>(w + h * v + j, k);
#pragma unroll
    for (int e = 0; e < VEC; ++e) a[e] = a[e] * inv * k[e] * sigmoid_f(c[e]);
    stv<T, VEC>(dst + j, a);
  }
}

}  // namespace

hipError_t lfmq_add_norm(void* x, const void* y, const void* w, float bias,
                         void* h, int n, int width, float eps, const void* wp,
                         const void* bp, void* p, int np, bool f32,
                         hipStream_t stream) {
  // rows per workgroup: 4 once the chip is full, else the row is shared
  const bool shared = n < 2048 || (u64)width * 16 > 64 * 1024;
  if ((u64)width * 4 > 64 * 1024) return hipErrorInvalidValue;
  const int rpw = shared ? 1 : 4;
  const int tpb = shared ? (width >= 2048 ? 512 : 256) : 256;
  const dim3 grid((n + rpw - 1) / rpw), block(tpb);
  const size_t lds = (size_t)rpw * width * sizeof(float);
#define GO(T, V, S)                                                          \
  hipLaunchKernelGGL((add_norm_kernel<T, V, S>), grid, block, lds, stream,   \
                     (float*)x, (const T*)y, (const float*)w, bias, (T*)h,   \
                     n, width, eps, (const T*)wp, (const float*)bp,          \
                     (float*)p, np)
#define GO2(T)                                                               \
  do {                                                                       \
    if (width % 4 == 0) {                                                    \
      if (shared) GO(T, 4, true); else GO(T, 4, false);                      \
    } else {                                                                 \
      if (shared) GO(T, 1, true); else GO(T, 1, false);                      \
    }                                                                        \
  } while (0)
  if (f32) GO2(float); else GO2(bf16_t);
#undef GO2
#undef GO
  return hipGetLastError();
}

hipError_t lfmq_head_norm_gate(const void* o, const void* g, long ldg,
                               const void* w, void* out, long rows, int heads,
                               int v, float eps, bool f32,
                               hipStream_t stream) {
  const u64 pairs = (u64)rows * heads;
  const dim3 grid((u32)((pairs + 3) / 4)), block(256);
  const bool v4 = v % 4 == 0 && ldg % 4 == 0 &&
                  (((u64)o | (u64)g | (u64)w | (u64)out) & 15) == 0;
#define GO(T, V)                                                             \
  hipLaunchKernelGGL((head_norm_gate_kernel<T, V>), grid, block, 0, stream,  \
                     (const float*)o, (const T*)g, (u64)ldg,                 \
                     (const float*)w, (T*)out, pairs, heads, v, eps)
  if (f32) { if (v4) GO(float, 4); else GO(float, 1); }
  else { if (v4) GO(bf16_t, 4); else GO(bf16_t, 1); }
#undef GO
  return hipGetLastError();
}
