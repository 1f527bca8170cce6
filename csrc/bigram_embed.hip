// Token embedding plus a hashed bigram embedding, into the fp32 residual
// stream:  x[row] = embed[tok] + bigram[hash(prev, tok)], with
// hash = (prev * mul_prev + tok * mul_cur) mod buckets, and the table's
// row `buckets` where a sequence has no previous token.  The token before
// a step's first one is part of the sequence's state (prev[slot]).
// seq_advance closes a step: lengths, previous tokens and the turn of the
// double-buffered recurrent vectors move on, all on the device, so that a
// decode step can be captured in a hipGraph.
#include "seq_common.h"

namespace {

template <typename T>
__global__ __launch_bounds__(256) void bigram_embed_kernel(
    const long* __restrict__ tok, SeqView sv, const i32* __restrict__ prev,
    const T* __restrict__ embed, const T* __restrict__ bigram,
    float* __restrict__ x, int width, long vocab, long buckets, long mul_prev,
    long mul_cur) {
  const int row = blockIdx.x;
  const int s = sv.seq[row];
  const int slot = sv.slots[s];
  long t = tok[row];
  t = t < 0 ? 0 : (t >= vocab ? vocab - 1 : t);  // the host validates ids
  const bool first = row == sv.cu[s];
  long p = -1;
  if (!first) p = tok[row - 1];
  else if (sv.lens[slot] > 0) p = prev[slot];
  const long r = p < 0 ? buckets : (p * mul_prev + t * mul_cur) % buckets;
  const T* e = embed + t * width;
  const T* g = bigram + r * width;
  for (int j = threadIdx.x; j < width; j += blockDim.x)
    x[(u64)row * width + j] = ldf(e + j) + ldf(g + j);
}

__global__ void seq_advance_kernel(const long* __restrict__ tok,
                                   const i32* __restrict__ cu,
                                   const i32* __restrict__ slots,
                                   i32* __restrict__ lens,
                                   i32* __restrict__ prev,
                                   i32* __restrict__ turn, int b) {
  const int s = blockIdx.x * blockDim.x + threadIdx.x;
  if (s >= b) return;
  const int n = cu[s + 1] - cu[s];
  if (n <= 0) return;
  const int slot = slots[s];
  prev[slot] = (i32)tok[cu[s + 1] - 1];
  lens[slot] += n;
  turn[slot] ^= 1;
}

}  // namespace

hipError_t lfmq_bigram_embed(const void* tok, const SeqView& sv,
                             const void* prev, const void* embed,
                             const void* bigram, void* x, int width,
                             long vocab, long buckets, long mul_prev,
                             long mul_cur, bool f32, hipStream_t stream) {
  if (buckets <= 0) return hipErrorInvalidValue;
#define GO(T)                                                                \
  hipLaunchKernelGGL(bigram_embed_kernel<T>, dim3(sv.n), dim3(256), 0,       \
                     stream, (const long*)tok, sv, (const i32*)prev,         \
                     (const T*)embed, (const T*)bigram, (float*)x, width,    \
                     vocab, buckets, mul_prev, mul_cur)
  if (f32) GO(float); else GO(bf16_t);
#undef GO
  return hipGetLastError();
}

hipError_t lfmq_seq_advance(const void* tok, const void* cu,
                            const void* slots, void* lens, void* prev,
                            void* turn, int b, hipStream_t stream) {
  hipLaunchKernelGGL(seq_advance_kernel, dim3((b + 63) / 64), dim3(64), 0,
                     stream, (const long*)tok, (const i32*)cu,
                     (const i32*)slots, (i32*)lens, (i32*)prev, (i32*)turn,
                     b);
  return hipGetLastError();
}
