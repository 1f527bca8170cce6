// Log gates of the mLSTM from their raw projections: both are soft-capped
// to (-cap, cap); the forget gate is a log-sigmoid on top.
#pragma once
#include <hip/hip_runtime.h>

__device__ __forceinline__ float mlstm_input_gate(float raw, float cap) {
  return cap * tanhf(raw / cap);
}
__device__ __forceinline__ float mlstm_forget_gate(float raw, float cap) {
  const float z = cap * tanhf(raw / cap);
  return fminf(z, 0.f) - log1pf(expf(-fabsf(z)));
}
