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

// C columns and EPT rows of the slice a thread; lanes run over the columns
// first, so that the sum over rows is a few shuffles and one LDS pass
template <typename T, int EPT, int C>
__global__ __launch_bounds__(TPB) void mlstm_scan_kernel(
    const T* __restrict__ qkv, u64 ld, const float* __restrict__ gates,
    SeqView sv, const i32* __restrict__ turn, float* __restrict__ S,
    float* __restrict__ nm, float* __restrict__ out, int heads, int dim,
    int vdim, float cap, int lanes_log2) {
  extern __shared__ float sh[];
  const int VL = 1 << lanes_log2;            // threads across the slice
  const int VS = VL * C, DG = TPB >> lanes_log2;
  float* qs = sh;                 // [2][dim]
  float* ks = sh + 2 * dim;       // [2][dim]
  float* red = sh + 4 * dim;      // [4 waves][VS]
  float* redn = red + 4 * VS;     // [4]
  const int s = blockIdx.z, h = blockIdx.y;
  const int n0 = sv.cu[s], n1 = sv.cu[s + 1];
  if (n1 <= n0) return;
  const int slot = sv.slots[s];
  const bool fresh = sv.lens[slot] == 0;
  const int cur = turn[slot] & 1;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int vl = threadIdx.x & (VL - 1), dg = threadIdx.x >> lanes_log2;
  const int v = blockIdx.x * VS + vl * C;    // C divides vdim
  const bool vok = v < vdim;
  const u64 sh_base = ((u64)slot * heads + h) * dim;
  float* Sp = S + sh_base * vdim;
  const float* nm_in = nm + (((u64)slot * 2 + cur) * heads + h) * (dim + 1);
  float* nm_out = nm + (((u64)slot * 2 + (cur ^ 1)) * heads + h) * (dim + 1);

  float st[EPT][C], nn[EPT];
#pragma unroll
  for (int e = 0; e < EPT; ++e) {
    const int d = dg + DG * e;
    if (!fresh && d < dim && vok) {
      ldv<float, C>(Sp + (u64)d * vdim + v, st[e]);
    } else {
#pragma unroll
      for (int c = 0; c < C; ++c) st[e][c] = 0.f;
    }
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
    float vv[C];
#pragma unroll
    for (int c = 0; c < C; ++c) vv[c] = vok ? ldf(r + voff + v + c) : 0.f;
    const float gi = mlstm_input_gate(gates[(u64)row * 2 * heads + h], cap);
    const float gf =
        mlstm_forget_gate(gates[(u64)row * 2 * heads + heads + h], cap);
    const float m2 = fmaxf(gf + m, gi);
    const float a = expf(gf + m - m2), b = expf(gi - m2);
    m = m2;
    __syncthreads();   // q, k staged; the last token's red is consumed
    float acc[C] = {}, den = 0.f;
#pragma unroll
    for (int e = 0; e < EPT; ++e) {
      const int d = dg + DG * e;
      const bool ok = d < dim;
      const float kd = ok ? k[d] : 0.f, qd = ok ? q[d] : 0.f;
      const float bk = b * kd;
#pragma unroll
      for (int c = 0; c < C; ++c) {
        st[e][c] = fmaf(a, st[e][c], bk * vv[c]);
        acc[c] = fmaf(st[e][c], qd, acc[c]);
      }
      nn[e] = fmaf(a, nn[e], bk);
      den = fmaf(nn[e], qd, den);
    }
    for (int o = VL; o < 64; o <<= 1) {
#pragma unroll
      for (int c = 0; c < C; ++c) acc[c] += __shfl_xor(acc[c], o, 64);
      den += __shfl_xor(den, o, 64);
    }
    if (lane < VL) {
#pragma unroll
      for (int c = 0; c < C; ++c) red[wave * VS + lane * C + c] = acc[c];
    }
    if (lane == 0) redn[wave] = den;
    __syncthreads();
    const int vo = blockIdx.x * VS + threadIdx.x;
    if (threadIdx.x < VS && vo < vdim) {
      float num = 0.f;
#pragma unroll
      for (int w = 0; w < TPB / 64; ++w) num += red[w * VS + threadIdx.x];
      const float dn = redn[0] + redn[1] + redn[2] + redn[3];
      out[((u64)row * heads + h) * vdim + vo] =
          num / (fmaxf(fabsf(dn), expf(-m)) + 1e-6f);
    }
  }
#pragma unroll
  for (int e = 0; e < EPT; ++e) {
    const int d = dg + DG * e;
    if (d < dim && vok) stv<float, C>(Sp + (u64)d * vdim + v, st[e]);
    if (d < dim && vl == 0 && blockIdx.x == 0) nm_out[d] = nn[e];
  }
  if (threadIdx.x == 0 && blockIdx.x == 0) nm_out[dim] = m;
}

}  // namespace

hipError_t lfmq_mlstm_scan(const void* qkv, long ld, const void* gates,
                           const SeqView& sv, const void* turn, void* S,
                           void* nm, void* out, int heads, int dim, int vdim,
                           float cap, bool f32, hipStream_t stream) {
  const int c = vdim % 4 == 0 ? 4 : 1;
  const int max_ept = c == 4 ? 16 : 64;
  // narrow slices give more workgroups, wide ones longer rows
  int vs = 64;
  while (vs > 16 &&
         ((u64)sv.b * heads * ((vdim + vs - 1) / vs) < 1024 ||
          dim > TPB * c / vs * max_ept))
    vs /= 2;
  int lanes_log2 = 0;
  while ((c << lanes_log2) < vs) ++lanes_log2;
  const int dg = TPB >> lanes_log2;
  const int ept = (dim + dg - 1) / dg;
  if (ept > max_ept) return hipErrorInvalidValue;
  const dim3 grid((vdim + vs - 1) / vs, heads, sv.b), block(TPB);
  const size_t lds = (4 * (size_t)dim + 4 * vs + 4) * sizeof(float);
#define GO(T, E, C)                                                          \
  hipLaunchKernelGGL((mlstm_scan_kernel<T, E, C>), grid, block, lds, stream, \
                     (const T*)qkv, (u64)ld, (const float*)gates, sv,        \
                     (const i32*)turn, (float*)S, (float*)nm, (float*)out,   \
                     heads, dim, vdim, cap, lanes_log2)
#define GO2(T)                                                               \
  do {                                                                       \
    if (c == 4) {                                                            \
      if (ept <= 1) GO(T, 1, 4);                                             \
      else if (ept <= 2) GO(T, 2, 4);                                        \
      else if (ept <= 4) GO(T, 4, 4);                                        \
      else if (ept <= 8) GO(T, 8, 4);                                        \
      else GO(T, 16, 4);                                                     \
    } else {                                                                 \
      if (ept <= 8) GO(T, 8, 1);                                             \
      else if (ept <= 16) GO(T, 16, 1);                                      \
      else GO(T, 64, 1);                                                     \
    }                                                                        \
  } while (0)
  if (f32) GO2(float); else GO2(bf16_t);
#undef GO2
#undef GO
  return hipGetLastError();
}
