// Shared device helpers of the sequence-mixing kernels (lfmq_seq).
//
// Batches are PACKED: a step brings N token rows of b sequences, without
// padding.  SeqView says which sequence a row belongs to, where each
// sequence's rows start, which cache slot it lives in and how many tokens
// the slot held before this step.  Every kernel is templated on the
// storage type T (bf16 or float); arithmetic is fp32 in both.
#pragma once
#include "common.h"

struct SeqView {
  const i32* seq;    // [N]   sequence of a row
  const i32* cu;     // [b+1] first row of a sequence
  const i32* slots;  // [b]   cache slot of a sequence
  const i32* lens;   // [slots] tokens in the slot before this step
  int b, n;
};

__device__ __forceinline__ float ldf(const float* p) { return *p; }
__device__ __forceinline__ float ldf(const bf16_t* p) {
  return bf16_bits_to_f32(*(const unsigned short*)p);
}
__device__ __forceinline__ void stf(float* p, float v) { *p = v; }
__device__ __forceinline__ void stf(bf16_t* p, float v) {
  *(unsigned short*)p = (unsigned short)f32_to_bf16_bits_rne(v);
}

typedef u32 u32x2 __attribute__((ext_vector_type(2)));

// four consecutive elements (the caller guarantees 4-element alignment)
__device__ __forceinline__ void ldf4(const float* p, float v[4]) {
  const f32x4 t = *(const f32x4*)p;
  v[0] = t[0]; v[1] = t[1]; v[2] = t[2]; v[3] = t[3];
}
__device__ __forceinline__ void ldf4(const bf16_t* p, float v[4]) {
  const u32x2 t = *(const u32x2*)p;
  bf16x2_to_f32(t[0], v[0], v[1]);
  bf16x2_to_f32(t[1], v[2], v[3]);
}
__device__ __forceinline__ void stf4(float* p, const float v[4]) {
  f32x4 t = {v[0], v[1], v[2], v[3]};
  *(f32x4*)p = t;
}
__device__ __forceinline__ void stf4(bf16_t* p, const float v[4]) {
  u32x2 t = {pack_bf16x2(v[0], v[1]), pack_bf16x2(v[2], v[3])};
  *(u32x2*)p = t;
}

template <typename T, int VEC>
__device__ __forceinline__ void ldv(const T* p, float v[VEC]) {
  if constexpr (VEC == 4) ldf4(p, v);
  else v[0] = ldf(p);
}
template <typename T, int VEC>
__device__ __forceinline__ void stv(T* p, const float v[VEC]) {
  if constexpr (VEC == 4) stf4(p, v);
  else stf(p, v[0]);
}

__device__ __forceinline__ float sigmoid_f(float x) {
  return 1.f / (1.f + expf(-x));
}

// split an fp32 value into two bf16 addends (16 significand bits): two
// MFMAs on the parts keep a 32-bit operand's precision
__device__ __forceinline__ void split_bf16(float x, unsigned short& hi,
                                           unsigned short& lo) {
  const u32 h = f32_to_bf16_bits_rne(x);
  hi = (unsigned short)h;
  lo = (unsigned short)f32_to_bf16_bits_rne(x - bf16_bits_to_f32(h));
}
