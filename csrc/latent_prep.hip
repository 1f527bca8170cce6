// Latent attention around the score kernels (attn_window*.hip).
//
// latent_prep: one pass over the fused input projection
//   [ query latent (q_rank) | kv latent (rank) | rotated key (rot) | ... ]
// norms both latents, rotates the shared key part, and writes the query
// latent plus the cache row {c [rank], k_rot [rot]} — straight into the
// ring cache for single-token steps, into the step's key buffer for
// prompts.
//
// The cache keeps the last `cap` tokens of a sequence: position p lives in
// ring row p mod cap.  latent_ring_load copies the cached tokens that a
// portion's windows reach back to in front of its own rows;
// latent_ring_store writes a portion's last `cap` rows back.
//
// latent_absorb / latent_expand: small per-head products for decode.  The
// key up-projection moves to the query (q_abs = q_h W_uk,h, next to the
// rotated query part) so that scores read the latent cache itself, and the
// value up-projection to the output, where the partial softmax results of
// a split key range are merged, the sink joins the denominator and the
// sigmoid output gate is applied.
#include "seq_common.h"

namespace {

__device__ __forceinline__ void rope_pair(int pos, float f, float u, float v,
                                          float& a, float& b) {
  float s, c;
  sincosf((float)pos * f, &s, &c);
  a = u * c - v * s;
  b = v * c + u * s;
}

// two waves a row: wave 0 the query latent, wave 1 the cache row
template <typename T, int VEC>
__global__ __launch_bounds__(256) void latent_prep_kernel(
    const T* __restrict__ in, u64 ld, SeqView sv,
    const float* __restrict__ wq, const float* __restrict__ wkv,
    const float* __restrict__ inv_freq, T* __restrict__ cq,
    T* __restrict__ dst, const i32* __restrict__ dst_row, int cap, int q_rank,
    int rank, int rot, int rot_dims, float eps) {
  const int row = blockIdx.x * 2 + (threadIdx.x >> 7);
  if (row >= sv.n) return;
  const bool kv = (threadIdx.x >> 6) & 1;
  const int lane = threadIdx.x & 63;
  const T* src = in + (u64)row * ld + (kv ? q_rank : 0);
  const int len = kv ? rank : q_rank;
  const float* w = kv ? wkv : wq;
  T* o = cq + (u64)row * q_rank;
  int pos = 0;
  if (kv) {
    const int s = sv.seq[row];
    const int slot = sv.slots[s], at = row - sv.cu[s];
    pos = sv.lens[slot] + at;
    const u64 drow = dst_row != nullptr ? (u64)(dst_row[s] + at)
                                        : (u64)slot * cap + pos % cap;
    o = dst + drow * (rank + rot);
  }
  float ss = 0.f;
#pragma unroll 4
  for (int j = lane * VEC; j < len; j += 64 * VEC) {
    float a[VEC];
    ldv<T, VEC>(src + j, a);
#pragma unroll
    for (int e = 0; e < VEC; ++e) ss = fmaf(a[e], a[e], ss);
  }
  ss = wave_reduce_sum(ss);
  const float inv = 1.f / sqrtf(ss / (float)len + eps);
#pragma unroll 4
  for (int j = lane * VEC; j < len; j += 64 * VEC) {
    float a[VEC], g[VEC];
    ldv<T, VEC>(src + j, a);
    ldv<float, VEC>(w + j, g);
#pragma unroll
    for (int e = 0; e < VEC; ++e) a[e] = a[e] * inv * g[e];
    stv<T, VEC>(o + j, a);
  }
  if (!kv) return;
  const T* kr = src + rank;
  const int half = rot_dims / 2;
  for (int j = lane; j < half; j += 64) {
    float a, b;
    rope_pair(pos, inv_freq[j], ldf(kr + j), ldf(kr + half + j), a, b);
    stf(o + rank + j, a);
    stf(o + rank + half + j, b);
  }
  for (int j = rot_dims + lane; j < rot; j += 64) stf(o + rank + j, ldf(kr + j));
}

// LOAD: key-buffer rows before a sequence's own come from the ring.
// Otherwise the last min(count, cap) rows of its own go into it.
// T is the unit of copying, d the units in a row.
template <typename T, bool LOAD>
__global__ __launch_bounds__(64) void latent_ring_kernel(
    SeqView sv, const i32* __restrict__ own_row, const i32* __restrict__ prior,
    T* __restrict__ buf, T* __restrict__ ring, int cap, int d) {
  const int s = blockIdx.y;
  const int slot = sv.slots[s];
  const int len0 = sv.lens[slot], cnt = sv.cu[s + 1] - sv.cu[s];
  const int total = LOAD ? prior[s] : min(cnt, cap);
  for (int i = blockIdx.x; i < total; i += gridDim.x) {
    const int pos = LOAD ? len0 - total + i : len0 + cnt - total + i;
    T* b = buf + (u64)(own_row[s] + pos - len0) * d;
    T* r = ring + ((u64)slot * cap + pos % cap) * d;
    for (int j = threadIdx.x; j < d; j += 64) {
      if (LOAD) b[j] = r[j]; else r[j] = b[j];
    }
  }
}

constexpr int PTPB = 512, PW = PTPB / 64;   // per-head products

// acc[i][c] = sum_k x[k][i] w[k][col + c] over this wave's share of k, then
// over the waves through red [PW][NB][64 NC].  A lane has NC columns.
template <typename T, int NB, int NC>
__device__ __forceinline__ void head_product(const float* x, int kdim,
                                             const T* w, int ncol, int n,
                                             float* red) {
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  float acc[NB][NC] = {};
  if (n < ncol) {
    const T* wp = w + n;
#pragma unroll 8
    for (int k = wave; k < kdim; k += PW) {
      float wv[NC];
      const T* p = wp + (u64)k * ncol;
      if constexpr (NC == 2 && sizeof(T) == 2) {
        bf16x2_to_f32(*(const u32*)p, wv[0], wv[1]);
      } else {
#pragma unroll
        for (int c = 0; c < NC; ++c) wv[c] = ldf(p + c);
      }
#pragma unroll
      for (int i = 0; i < NB; ++i)
#pragma unroll
        for (int c = 0; c < NC; ++c)
          acc[i][c] = fmaf(x[k * NB + i], wv[c], acc[i][c]);
    }
  }
#pragma unroll
  for (int i = 0; i < NB; ++i)
#pragma unroll
    for (int c = 0; c < NC; ++c)
      red[((wave * NB + i) * NC + c) * 64 + lane] = acc[i][c];
  __syncthreads();
}

template <int NB, int NC>
__device__ __forceinline__ float head_sum(const float* red, int i, int c,
                                          int lane) {
  float v = 0.f;
#pragma unroll
  for (int g = 0; g < PW; ++g) v += red[((g * NB + i) * NC + c) * 64 + lane];
  return v;
}

// y[b, h, n] = sum_k q[b, h, k] W[h, k, n] for n < rank; rotated query
// part behind it.  NB sequences share a pass over the weights.
template <typename T, int NB, int NC>
__global__ __launch_bounds__(PTPB) void latent_absorb_kernel(
    const T* __restrict__ q, const T* __restrict__ w, SeqView sv,
    const float* __restrict__ inv_freq, T* __restrict__ out, int heads,
    int dim, int rot, int rot_dims, int rank) {
  extern __shared__ float sh[];
  float* x = sh;                     // [dim][NB]
  float* red = sh + NB * dim;        // [PW][NB][NC][64]
  const int h = blockIdx.y, b0 = blockIdx.z * NB;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int n = (blockIdx.x * 64 + lane) * NC;
  for (int i = threadIdx.x; i < NB * dim; i += PTPB) {
    const int bb = b0 + i / dim, k = i % dim;
    x[k * NB + i / dim] =
        bb < sv.b ? ldf(q + ((u64)bb * heads + h) * (dim + rot) + k) : 0.f;
  }
  __syncthreads();
  head_product<T, NB, NC>(x, dim, w + (u64)h * dim * rank, rank, n, red);
  for (int i = wave; i < NB; i += PW) {
    const int bb = b0 + i;
    if (bb >= sv.b) continue;
    T* o = out + ((u64)bb * heads + h) * (rank + rot);
    if (n < rank) {
#pragma unroll
      for (int c = 0; c < NC; ++c)
        stf(o + n + c, head_sum<NB, NC>(red, i, c, lane));
    }
    if (blockIdx.x == 0) {
      const T* qr = q + ((u64)bb * heads + h) * (dim + rot) + dim;
      const int pos = sv.lens[sv.slots[bb]];
      const int half = rot_dims / 2;
      for (int j = lane; j < half; j += 64) {
        float a, c;
        rope_pair(pos, inv_freq[j], ldf(qr + j), ldf(qr + half + j), a, c);
        stf(o + rank + j, a);
        stf(o + rank + half + j, c);
      }
      for (int j = rot_dims + lane; j < rot; j += 64)
        stf(o + rank + j, ldf(qr + j));
    }
  }
}

// part [b, splits, heads, rank + 2] = {sum p c, max, sum p} per key range
template <typename T, int NB, int NC>
__global__ __launch_bounds__(PTPB) void latent_expand_kernel(
    const float* __restrict__ part, int splits, const float* __restrict__ sink,
    const T* __restrict__ w, const T* __restrict__ g, u64 ldg,
    T* __restrict__ out, int b, int heads, int rank, int vdim) {
  extern __shared__ float sh[];
  float* x = sh;                     // [rank][NB]
  float* red = x + NB * rank;        // [PW][NB][NC][64]
  float* wt = red + PW * NB * NC * 64;   // [NB][splits]
  const int h = blockIdx.y, b0 = blockIdx.z * NB;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int n = (blockIdx.x * 64 + lane) * NC;
  const u64 pr = rank + 2, sp = (u64)heads * pr;
  // weight of every key range: the sink joins maximum and denominator
  for (int i = wave; i < NB; i += PW) {
    if (b0 + i >= b) continue;
    const float* p = part + ((u64)(b0 + i) * splits * heads + h) * pr + rank;
    float M = sink[h];
    for (int c = lane; c < splits; c += 64) M = fmaxf(M, p[c * sp]);
    M = wave_reduce_max(M);
    float L = 0.f;
    for (int c = lane; c < splits; c += 64) {
      const float e = expf(p[c * sp] - M);
      wt[i * splits + c] = e;
      L = fmaf(e, p[c * sp + 1], L);
    }
    L = wave_reduce_sum(L) + expf(sink[h] - M);
    for (int c = lane; c < splits; c += 64) wt[i * splits + c] /= L;
  }
  __syncthreads();
  for (int id = threadIdx.x; id < NB * rank; id += PTPB) {
    const int i = id / rank, j = id % rank;
    float a = 0.f;
    if (b0 + i < b) {
      const float* p = part + ((u64)(b0 + i) * splits * heads + h) * pr + j;
#pragma unroll 8
      for (int c = 0; c < splits; ++c)
        a = fmaf(wt[i * splits + c], p[c * sp], a);
    }
    x[j * NB + i] = a;
  }
  __syncthreads();
  head_product<T, NB, NC>(x, rank, w + (u64)h * rank * vdim, vdim, n, red);
  if (n >= vdim) return;
  for (int i = wave; i < NB; i += PW) {
    const int bb = b0 + i;
    if (bb >= b) continue;
#pragma unroll
    for (int c = 0; c < NC; ++c) {
      const u64 o = (u64)h * vdim + n + c;
      stf(out + (u64)bb * heads * vdim + o,
          head_sum<NB, NC>(red, i, c, lane) *
              sigmoid_f(ldf(g + (u64)bb * ldg + o)));
    }
  }
}

}  // namespace

hipError_t lfmq_latent_prep(const void* in, long ld, const SeqView& sv,
                            const void* wq, const void* wkv,
                            const void* inv_freq, void* cq, void* dst,
                            const void* dst_row, int cap, int q_rank,
                            int rank, int rot, int rot_dims, float eps,
                            bool f32, hipStream_t stream) {
  const dim3 grid((sv.n + 1) / 2), block(256);
  const bool v4 = ((ld | q_rank | rank | rot) & 3) == 0 &&
                  (((u64)in | (u64)dst | (u64)wq | (u64)wkv) & 15) == 0;
#define GO(T, V)                                                             \
  hipLaunchKernelGGL((latent_prep_kernel<T, V>), grid, block, 0, stream,     \
                     (const T*)in, (u64)ld, sv, (const float*)wq,            \
                     (const float*)wkv, (const float*)inv_freq, (T*)cq,      \
                     (T*)dst, (const i32*)dst_row, cap, q_rank, rank, rot,   \
                     rot_dims, eps)
  if (f32) { if (v4) GO(float, 4); else GO(float, 1); }
  else { if (v4) GO(bf16_t, 4); else GO(bf16_t, 1); }
#undef GO
  return hipGetLastError();
}

hipError_t lfmq_latent_ring(const SeqView& sv, const void* own_row,
                            const void* prior, void* buf, void* ring, int cap,
                            int d, bool load, bool f32, hipStream_t stream) {
  const dim3 grid(cap < 2048 ? cap : 2048, sv.b), block(64);
  const int bytes = d * (f32 ? 4 : 2);
#define GO(T, L)                                                             \
  hipLaunchKernelGGL((latent_ring_kernel<T, L>), grid, block, 0, stream, sv, \
                     (const i32*)own_row, (const i32*)prior, (T*)buf,        \
                     (T*)ring, cap, bytes / (int)sizeof(T))
#define GO2(T)                                                               \
  do {                                                                       \
    if (load) GO(T, true); else GO(T, false);                                \
  } while (0)
  if (bytes % 16 == 0 && (((u64)buf | (u64)ring) & 15) == 0) GO2(u32x4);
  else if (bytes % 4 == 0) GO2(u32);
  else GO2(unsigned short);
#undef GO2
#undef GO
  return hipGetLastError();
}

// as many sequences as there are and LDS has room for
static int sequences_per_pass(int b, int nc, int per_seq) {
  int nb = b == 1 ? 1 : (b <= 4 ? 4 : 8);
  while (nb > 1 && (size_t)nb * (per_seq + PW * nc * 64) * 4 > 64 * 1024)
    nb = nb == 8 ? 4 : 1;
  return nb;
}

// NB sequences and NC columns a lane, by batch and width
#define LFMQ_HEAD_PRODUCT(T)                                                 \
  do {                                                                       \
    if (nc == 2) {                                                           \
      if (nb == 1) GO(T, 1, 2); else if (nb == 4) GO(T, 4, 2);               \
      else GO(T, 8, 2);                                                      \
    } else {                                                                 \
      if (nb == 1) GO(T, 1, 1); else if (nb == 4) GO(T, 4, 1);               \
      else GO(T, 8, 1);                                                      \
    }                                                                        \
  } while (0)

hipError_t lfmq_latent_absorb(const void* q, const void* w, const SeqView& sv,
                              const void* inv_freq, void* out, int heads,
                              int dim, int rot, int rot_dims, int rank,
                              bool f32, hipStream_t stream) {
  const int nc = rank % 2 == 0 ? 2 : 1;
  const int nb = sequences_per_pass(sv.b, nc, dim);
  const dim3 grid((rank + 64 * nc - 1) / (64 * nc), heads,
                  (sv.b + nb - 1) / nb), block(PTPB);
  const size_t lds = (nb * (size_t)dim + PW * nb * nc * 64) * sizeof(float);
  if (lds > 64 * 1024) return hipErrorInvalidValue;
#define GO(T, B, C)                                                          \
  hipLaunchKernelGGL((latent_absorb_kernel<T, B, C>), grid, block, lds,      \
                     stream, (const T*)q, (const T*)w, sv,                   \
                     (const float*)inv_freq, (T*)out, heads, dim, rot,       \
                     rot_dims, rank)
  if (f32) LFMQ_HEAD_PRODUCT(float); else LFMQ_HEAD_PRODUCT(bf16_t);
#undef GO
  return hipGetLastError();
}

hipError_t lfmq_latent_expand(const void* part, int splits, const void* sink,
                              const void* w, const void* g, long ldg,
                              void* out, int b, int heads, int rank, int vdim,
                              bool f32, hipStream_t stream) {
  const int nc = vdim % 2 == 0 ? 2 : 1;
  const int nb = sequences_per_pass(b, nc, rank + splits);
  const dim3 grid((vdim + 64 * nc - 1) / (64 * nc), heads, (b + nb - 1) / nb),
      block(PTPB);
  const size_t lds = (nb * (size_t)rank + PW * nb * nc * 64 +
                      nb * (size_t)splits) * sizeof(float);
  if (lds > 64 * 1024) return hipErrorInvalidValue;
#define GO(T, B, C)                                                          \
  hipLaunchKernelGGL((latent_expand_kernel<T, B, C>), grid, block, lds,      \
                     stream, (const float*)part, splits, (const float*)sink, \
                     (const T*)w, (const T*)g, (u64)ldg, (T*)out, b, heads,  \
                     rank, vdim)
  if (f32) LFMQ_HEAD_PRODUCT(float); else LFMQ_HEAD_PRODUCT(bf16_t);
#undef GO
  return hipGetLastError();
}
#undef LFMQ_HEAD_PRODUCT
