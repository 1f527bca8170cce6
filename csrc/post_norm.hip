// Norm on a sublayer's OUTPUT, added to the fp32 residual stream:
//   x += rms(y) * w,   h = x in the model's dtype
// or, with an output norm, h = rms(x) * w_out * gain (the model's last norm
// and its logit scale).  One pass over the row.
//
// y comes from one of
//   rows     a tensor [n, width]
//   table    embedding rows (x starts there: x = rms(table[tok]) * w)
//   experts  the sum of a token's `top` expert rows, plus a shared expert's
//            row times a number per token
//
// One wave owns a row; with few rows a whole workgroup shares one.
#include "seq_common.h"

namespace {

enum Source { ROWS, TABLE, EXPERTS };

struct PostArgs {
  float* x;
  const void* y;          // rows, table, or expert rows
  const int64_t* tok;     // TABLE
  const i32* pos;         // EXPERTS: [n, top] rows of y
  const void* shared;     // EXPERTS: [n, width] or null
  const float* sgate;     // EXPERTS: [n]
  const float* w;
  const float* w_out;     // or null
  void* h;                // or null
  int n, width, top, vocab;
  float eps, gain;
};

template <typename T, int VEC, bool SHARED, int SRC>
__global__ __launch_bounds__(512) void post_norm_kernel(PostArgs A) {
  extern __shared__ float rows[];
  __shared__ float red[2][8];
  const int wave = threadIdx.x / LFMQ_WAVE, lane = threadIdx.x % LFMQ_WAVE;
  const int nwave = blockDim.x / LFMQ_WAVE;
  constexpr int rpw = SHARED ? 1 : 4;
  const int lr = SHARED ? 0 : wave;
  const int row = blockIdx.x * rpw + lr;
  const int t0 = (SHARED ? threadIdx.x : lane) * VEC;
  const int step = (SHARED ? blockDim.x : LFMQ_WAVE) * VEC;
  const int width = A.width;
  const bool live = row < A.n;
  float* hr = rows + (u64)lr * width;
  float* xr = A.x + (u64)row * width;
  T* out = (T*)A.h + (u64)row * width;

  auto total = [&](float v, int which) {
    v = wave_reduce_sum(v);
    if constexpr (SHARED) {
      if (lane == 0) red[which][wave] = v;
      __syncthreads();
      v = 0.f;
      for (int i = 0; i < nwave; ++i) v += red[which][i];
    }
    return v;
  };

  float ss = 0.f;
  if (live) {
    const T* src = (const T*)A.y;
    if constexpr (SRC == ROWS) src += (u64)row * width;
    if constexpr (SRC == TABLE) {
      const int64_t t = A.tok[row];
      src += (u64)(t < 0 ? 0 : (t >= A.vocab ? A.vocab - 1 : t)) * width;
    }
    constexpr int PK = 8;           // choices kept in registers
    u64 at[PK] = {};
    if constexpr (SRC == EXPERTS) {
#pragma unroll
      for (int k = 0; k < PK; ++k)
        if (k < A.top) at[k] = (u64)A.pos[(u64)row * A.top + k] * width;
    }
    const float sg =
        SRC == EXPERTS && A.shared != nullptr ? A.sgate[row] : 0.f;
    for (int j = t0; j < width; j += step) {
      float a[VEC];
      if constexpr (SRC == EXPERTS) {
#pragma unroll
        for (int e = 0; e < VEC; ++e) a[e] = 0.f;
#pragma unroll
        for (int k = 0; k < PK; ++k) {
          if (k >= A.top) break;
          float c[VEC];
          ldv<T, VEC>(src + at[k] + j, c);
#pragma unroll
          for (int e = 0; e < VEC; ++e) a[e] += c[e];
        }
        for (int k = PK; k < A.top; ++k) {
          float c[VEC];
          ldv<T, VEC>(src + (u64)A.pos[(u64)row * A.top + k] * width + j, c);
#pragma unroll
          for (int e = 0; e < VEC; ++e) a[e] += c[e];
        }
        if (A.shared != nullptr) {
          float c[VEC];
          ldv<T, VEC>((const T*)A.shared + (u64)row * width + j, c);
#pragma unroll
          for (int e = 0; e < VEC; ++e) a[e] = fmaf(sg, c[e], a[e]);
        }
      } else {
        ldv<T, VEC>(src + j, a);
      }
#pragma unroll
      for (int e = 0; e < VEC; ++e) ss = fmaf(a[e], a[e], ss);
      stv<float, VEC>(hr + j, a);
    }
  }
  const float inv = 1.f / sqrtf(total(ss, 0) / (float)width + A.eps);
  ss = 0.f;
  if (live) {
    // every thread takes the very elements that it stored
    for (int j = t0; j < width; j += step) {
      float a[VEC], g[VEC];
      ldv<float, VEC>(hr + j, a);
      ldv<float, VEC>(A.w + j, g);
#pragma unroll
      for (int e = 0; e < VEC; ++e) a[e] = a[e] * inv * g[e];
      if constexpr (SRC != TABLE) {
        float o[VEC];
        ldv<float, VEC>(xr + j, o);
#pragma unroll
        for (int e = 0; e < VEC; ++e) a[e] += o[e];
      }
      stv<float, VEC>(xr + j, a);
      if (A.w_out != nullptr) {
#pragma unroll
        for (int e = 0; e < VEC; ++e) ss = fmaf(a[e], a[e], ss);
        stv<float, VEC>(hr + j, a);
      } else if (A.h != nullptr) {
        stv<T, VEC>(out + j, a);
      }
    }
  }
  if (A.w_out == nullptr) return;
  const float inv2 = 1.f / sqrtf(total(ss, 1) / (float)width + A.eps);
  if (!live) return;
  for (int j = t0; j < width; j += step) {
    float a[VEC], g[VEC];
    ldv<float, VEC>(hr + j, a);
    ldv<float, VEC>(A.w_out + j, g);
#pragma unroll
    for (int e = 0; e < VEC; ++e) a[e] = a[e] * inv2 * g[e] * A.gain;
    stv<T, VEC>(out + j, a);
  }
}

template <typename T, int SRC>
void launch(const PostArgs& A, hipStream_t stream) {
  // four rows a workgroup once the chip is full, else the row is shared
  const bool shared = A.n < 2048 || (u64)A.width * 16 > 64 * 1024;
  const int rpw = shared ? 1 : 4;
  const int tpb = shared && A.width >= 2048 ? 512 : 256;
  const dim3 grid((A.n + rpw - 1) / rpw), block(tpb);
  const size_t lds = (size_t)rpw * A.width * sizeof(float);
  const bool v4 =
      A.width % 4 == 0 &&
      (((u64)A.x | (u64)A.y | (u64)A.shared | (u64)A.w | (u64)A.w_out |
        (u64)A.h) & 15) == 0;
#define GO(V, S)                                                             \
  hipLaunchKernelGGL((post_norm_kernel<T, V, S, SRC>), grid, block, lds,     \
                     stream, A)
  if (v4) { if (shared) GO(4, true); else GO(4, false); }
  else { if (shared) GO(1, true); else GO(1, false); }
#undef GO
}

template <int SRC>
hipError_t go(const PostArgs& A, bool f32, hipStream_t stream) {
  if ((u64)A.width * 4 > 64 * 1024) return hipErrorInvalidValue;
  if (f32) launch<float, SRC>(A, stream);
  else launch<bf16_t, SRC>(A, stream);
  return hipGetLastError();
}

}  // namespace

hipError_t lfmq_post_norm(void* x, const void* y, const void* w,
                          const void* w_out, void* h, int n, int width,
                          float eps, float gain, bool f32,
                          hipStream_t stream) {
  PostArgs A{(float*)x, y, nullptr, nullptr, nullptr, nullptr,
             (const float*)w, (const float*)w_out, h, n, width, 0, 0, eps,
             gain};
  return go<ROWS>(A, f32, stream);
}

hipError_t lfmq_embed_norm(void* x, const void* table, const void* tok,
                           const void* w, void* h, int n, int width,
                           int vocab, float eps, bool f32,
                           hipStream_t stream) {
  PostArgs A{(float*)x, table, (const int64_t*)tok, nullptr, nullptr, nullptr,
             (const float*)w, nullptr, h, n, width, 0, vocab, eps, 1.f};
  return go<TABLE>(A, f32, stream);
}

hipError_t lfmq_post_norm_experts(void* x, const void* rows, const void* pos,
                                  int top, const void* shared,
                                  const void* sgate, const void* w,
                                  const void* w_out, void* h, int n,
                                  int width, float eps, float gain, bool f32,
                                  hipStream_t stream) {
  PostArgs A{(float*)x, rows, nullptr, (const i32*)pos, shared,
             (const float*)sgate, (const float*)w, (const float*)w_out, h, n,
             width, top, 0, eps, gain};
  return go<EXPERTS>(A, f32, stream);
}
