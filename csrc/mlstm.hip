// Matrix-memory LSTM (mLSTM) — token recurrence.
//
// Per head, with log gates i (input) and f (forget) and a running maximum
// m that starts at 0:
//   m' = max(f + m, i)
//   S' = exp(f + m - m') S + exp(i - m') k v^T      n' likewise, v = 1
//   o  = S'^T q / (max(|n' . q|, exp(-m')) + 1e-6)
// State in fp32: S [slots, H, dim, vdim]; the vectors {n [dim], m} are
// double-buffered [slots, 2, H, dim + 1] and `turn[slot]` names the buffer
// to read — every workgroup of a head needs all of n, so the one that
// writes the new n must not touch what its neighbours still read.  A slot
// of length 0 starts from zeros whatever it holds.
//
// mlstm_scan runs any number of tokens per sequence one by one: decode
// (memory-bound, one state read and write), 32-bit prompts and short
// portions.  Grid (vdim / VS, heads, sequences); a workgroup keeps its
// [dim x VS] slice of S in registers.  mlstm_chunk.hip is the MFMA form
// for 16-bit prompts.
#include "seq_common.h"

#include "mlstm_gate.h"

namespace {

constexpr int TPB = 256;

template <typename T, int EPT>
__global__ __launch_bounds__(TPB) void mlstm_scan_kernel(
    const T* __restrict__ qkv, u64 ld, const float* __restrict__ gates,
    SeqView sv, const i32* __restrict__ turn, float* __restrict__ S,
    float* __restrict__ nm, float* __restrict__ out, int heads, int dim,
    int vdim, float cap, int vs_log2) {
  extern __shared__ float sh[];
  const int VS = 1 << vs_log2;
  const int DG = TPB >> vs_log2;
  float* qs = sh;                 // [2][dim]
  float* ks = sh + 2 * dim;       // [2][dim]
  float* red = sh + 4 * dim;      // [TPB]
  float* redn = red + TPB;        // [DG]
  const int s = blockIdx.z, h = blockIdx.y;
  const int n0 = sv.cu[s], n1 = sv.cu[s + 1];
  if (n1 <= n0) return;
  const int slot = sv.slots[s];
  const bool fresh = sv.lens[slot] == 0;
  const int cur = turn[slot] & 1;
  const int vl = threadIdx.x & (VS - 1), dg = threadIdx.x >> vs_log2;
  const int v = blockIdx.x * VS + vl;
  const bool vok = v < vdim;
  const u64 sh_base = ((u64)slot * heads + h) * dim;
  float* Sp = S + sh_base * vdim;
  const float* nm_in = nm + (((u64)slot * 2 + cur) * heads + h) * (dim + 1);
  float* nm_out = nm + (((u64)slot * 2 + (cur ^ 1)) * heads + h) * (dim + 1);

  float st[EPT], nn[EPT];
#pragma unroll
  for (int e = 0; e < EPT; ++e) {
    const int d = dg + DG * e;
    st[e] = (!fresh && d < dim && vok) ? Sp[(u64)d * vdim + v] : 0.f;
    nn[e] = (!fresh && d < dim) ? nm_in[d] : 0.f;
  }
  float m = fresh ? 0.f : nm_in[dim];
  const float qscale = 1.f / sqrtf((float)dim);
  const T* base = qkv + (u64)h * dim;
  const u64 koff = (u64)heads * dim;
  const u64 voff = 2 * koff + (u64)h * vdim - (u64)h * dim;

  for (int row = n0; row < n1; ++row) {
    const T* r = base + (u64)row * ld;
    float* q = qs + ((row - n0) & 1) * dim;
    float* k = ks + ((row - n0) & 1) * dim;
    for (int d = threadIdx.x; d < dim; d += TPB) {
      q[d] = ldf(r + d) * qscale;
      k[d] = ldf(r + koff + d);
    }
    const float vv = vok ? ldf(r + voff + v) : 0.f;
    const float gi = mlstm_input_gate(gates[(u64)row * 2 * heads + h], cap);
    const float gf =
        mlstm_forget_gate(gates[(u64)row * 2 * heads + heads + h], cap);
    const float m2 = fmaxf(gf + m, gi);
    const float a = expf(gf + m - m2), b = expf(gi - m2);
    m = m2;
    __syncthreads();   // q, k staged; the last token's red is consumed
    float acc = 0.f, den = 0.f;
#pragma unroll
    for (int e = 0; e < EPT; ++e) {
      const int d = dg + DG * e;
      const bool ok = d < dim;
      const float kd = ok ? k[d] : 0.f, qd = ok ? q[d] : 0.f;
      st[e] = fmaf(a, st[e], b * kd * vv);
      nn[e] = fmaf(a, nn[e], b * kd);
      acc = fmaf(st[e], qd, acc);
      den = fmaf(nn[e], qd, den);
    }
    red[threadIdx.x] = acc;
    if (vl == 0) redn[dg] = den;
    __syncthreads();
    if (dg == 0 && vok) {
      float num = 0.f, dn = 0.f;
      for (int g = 0; g < DG; ++g) {
        num += red[g * VS + vl];
        dn += redn[g];
      }
      out[((u64)row * heads + h) * vdim + v] =
          num / (fmaxf(fabsf(dn), expf(-m)) + 1e-6f);
    }
  }
#pragma unroll
  for (int e = 0; e < EPT; ++e) {
    const int d = dg + DG * e;
    if (d < dim && vok) Sp[(u64)d * vdim + v] = st[e];
    if (d < dim && vl == 0 && blockIdx.x == 0) nm_out[d] = nn[e];
  }
  if (threadIdx.x == 0 && blockIdx.x == 0) nm_out[dim] = m;
}

}  // namespace

hipError_t lfmq_mlstm_scan(const void* qkv, long ld, const void* gates,
                           const SeqView& sv, const void* turn, void* S,
                           void* nm, void* out, int heads, int dim, int vdim,
                           float cap, bool f32, hipStream_t stream) {
  // narrow value slices give more workgroups; wide ones longer rows
  int vl = 6;
  while (vl > 4 && ((u64)sv.b * heads * ((vdim + (1 << vl) - 1) >> vl) < 1024 ||
                    dim > (TPB >> vl) * 64))
    --vl;
  const int dg = TPB >> vl;
  const int ept = (dim + dg - 1) / dg;
  if (ept > 64) return hipErrorInvalidValue;
  const dim3 grid((vdim + (1 << vl) - 1) >> vl, heads, sv.b), block(TPB);
  const size_t lds = (4 * (size_t)dim + TPB + dg) * sizeof(float);
#define GO(T, E)                                                             \
  hipLaunchKernelGGL((mlstm_scan_kernel<T, E>), grid, block, lds, stream,    \
                     (const T*)qkv, (u64)ld, (const float*)gates, sv,        \
                     (const i32*)turn, (float*)S, (float*)nm, (float*)out,   \
                     heads, dim, vdim, cap, vl)
#define GO2(T)                                                               \
  do {                                                                       \
    if (ept <= 4) GO(T, 4);                                                  \
    else if (ept <= 8) GO(T, 8);                                             \
    else if (ept <= 16) GO(T, 16);                                           \
    else if (ept <= 32) GO(T, 32);                                           \
    else GO(T, 64);                                                          \
  } while (0)
  if (f32) GO2(float); else GO2(bf16_t);
#undef GO2
#undef GO
  return hipGetLastError();
}
