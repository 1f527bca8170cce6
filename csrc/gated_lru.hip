// Real-gated linear recurrent unit behind a short causal convolution.
//   u = conv(x + xb) + cb                   per channel, zeros before token 0
//   r = sigmoid(Wr u + br), i = sigmoid(Wi u + bi)   block-diagonal
//   log a = c r softplus(lam),  z = sqrt(1 - a^2) i u
//   S = a S + z,   out = gain S gelu(y + yb)
// State: S fp32 [slots, C], and the convolution's last `taps` inputs fp32
// [slots, taps, C], where position p lives in row p mod taps (a token reads
// the other rows and writes its own, so that one step's workgroups do not
// meet).  A slot of length 0 starts from zeros whatever it holds.
//
// 16-bit prompts: lru_conv, then lru_gates on the matrix cores, whose
// epilogue already runs the recurrence inside tiles of 64 tokens (every
// token's {decay, state} relative to its tile's start), lru_carry over the
// tiles, lru_apply.  16-bit single tokens: lru_step does all of it at once.
// Any other size and 32-bit storage: lru_conv, lru_gates_any, lru_scan.
#include "seq_common.h"

namespace {

constexpr int TM = 64;      // tokens a tile
constexpr int KC = 256;     // gate inputs staged at a time (prompts)
constexpr int SKC = 512;    // the same, single tokens

struct LruArgs {
  const void *x, *y;        // projection columns, row stride ld
  u64 ld;
  const float *xb, *yb, *cw, *cb, *gb, *lam;   // cw [taps, C], gb [B, 2, n]
  const void* gw;           // [B, 2, n, n] rows = outputs
  float *ring, *S;
  void* out;
  u64 ldo;
  int C, blocks, n, taps;
  float c, gain;
  bool x4;                  // four columns of x may be loaded at once
};

__device__ __forceinline__ float softplus_f(float x) {
  return x > 20.f ? x : log1pf(expf(x));
}
// FAST: the hardware's exponential, reciprocal and root, each good to a few
// units in the last place (32-bit storage takes the library's)
template <bool FAST>
__device__ __forceinline__ float sigm(float x) {
  if constexpr (FAST) return __builtin_amdgcn_rcpf(1.f + __expf(-x));
  return sigmoid_f(x);
}
// 0.5 x (1 + tanh(t)) = x sigmoid(2 t)
template <bool FAST>
__device__ __forceinline__ float gelu_tanh_f(float x) {
  const float k = 0.7978845608028654f;
  return x * sigm<FAST>(2.f * k * fmaf(0.044715f * x * x, x, x));
}
// gate pre-activations and u -> decay and input.  1 - a^2 = -(e^t - 1) with
// t = 2 log a, by its series where the difference would cancel.
template <bool FAST>
__device__ __forceinline__ void lru_pair(float r, float i, float u, float csp,
                                         float& a, float& z) {
  const float la = csp * sigm<FAST>(r);
  if constexpr (FAST) {
    a = __expf(la);
    const float t = 2.f * la;
    float s = 1.f + t * (1.f / 8.f);
    s = fmaf(t * (1.f / 7.f), s, 1.f);
    s = fmaf(t * (1.f / 6.f), s, 1.f);
    s = fmaf(t * (1.f / 5.f), s, 1.f);
    s = fmaf(t * (1.f / 4.f), s, 1.f);
    s = fmaf(t * (1.f / 3.f), s, 1.f);
    s = fmaf(t * (1.f / 2.f), s, 1.f);
    const float d = t > -0.5f ? -t * s : fmaf(-a, a, 1.f);
    z = __builtin_amdgcn_sqrtf(d) * sigm<true>(i) * u;
  } else {
    a = expf(la);
    z = sqrtf(-expm1f(2.f * la)) * sigm<false>(i) * u;
  }
}
__device__ __forceinline__ float round_to(float v, const float*) { return v; }
__device__ __forceinline__ float round_to(float v, const bf16_t*) {
  return bf16_bits_to_f32(f32_to_bf16_bits_rne(v));
}

// convolution input of channel c, `back` tokens before `row`
template <typename T>
__device__ __forceinline__ float conv_in(const LruArgs& A, int row, int row0,
                                         int pos, int slot, int back, int c) {
  if (row - back >= row0)
    return ldf((const T*)A.x + (u64)(row - back) * A.ld + c) + A.xb[c];
  const int p = pos - back;
  return p >= 0 ? A.ring[((u64)slot * A.taps + p % A.taps) * A.C + c] : 0.f;
}
template <typename T>
__device__ __forceinline__ float conv_at(const LruArgs& A, int row, int row0,
                                         int pos, int slot, int c) {
  float v = A.cb[c];
  for (int j = 0; j < A.taps; ++j)
    v = fmaf(A.cw[(u64)j * A.C + c],
             conv_in<T>(A, row, row0, pos, slot, A.taps - 1 - j, c), v);
  return round_to(v, (const T*)nullptr);
}

template <typename T>
__device__ __forceinline__ void load_x4(const LruArgs& A, int row, int c,
                                        float v[4]) {
  const T* p = (const T*)A.x + (u64)row * A.ld + c;
  if (A.x4) {
    ldf4(p, v);
  } else {
#pragma unroll
    for (int e = 0; e < 4; ++e) v[e] = ldf(p + e);
  }
}

constexpr int RC = 8;       // consecutive rows of a thread

// u [n, C].  Four taps and C % 4 == 0: a thread takes four channels and
// keeps the last inputs in registers
template <typename T>
__global__ __launch_bounds__(256) void lru_conv4_kernel(SeqView sv, LruArgs A,
                                                        T* __restrict__ u) {
  const int c = (blockIdx.x * 256 + threadIdx.x) * 4;
  if (c >= A.C) return;
  const int r0 = blockIdx.y * RC, r1 = min(r0 + RC, sv.n);
  float w[4][4], in[4][4] = {}, b[4], xb[4], nx[RC][4];
#pragma unroll
  for (int j = 0; j < 4; ++j) ldf4(A.cw + (u64)j * A.C + c, w[j]);
  ldf4(A.cb + c, b);
  ldf4(A.xb + c, xb);
#pragma unroll
  for (int i = 0; i < RC; ++i)
    if (r0 + i < r1) load_x4<T>(A, r0 + i, c, nx[i]);
  int last = -1;
#pragma unroll
  for (int i = 0; i < RC; ++i) {
    const int row = r0 + i;
    if (row >= r1) break;
    const int s = sv.seq[row];
    if (s != last) {        // the three inputs before this one
      const int slot = sv.slots[s], row0 = sv.cu[s];
      const int pos = sv.lens[slot] + row - row0;
#pragma unroll
      for (int j = 1; j < 4; ++j)
#pragma unroll
        for (int e = 0; e < 4; ++e)
          in[4 - j][e] = conv_in<T>(A, row, row0, pos, slot, j, c + e);
      last = s;
    }
    float v[4];
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      in[0][e] = in[1][e];
      in[1][e] = in[2][e];
      in[2][e] = in[3][e];
      in[3][e] = nx[i][e] + xb[e];
      v[e] = b[e];
#pragma unroll
      for (int j = 0; j < 4; ++j) v[e] = fmaf(w[j][e], in[j][e], v[e]);
    }
    stf4(u + (u64)row * A.C + c, v);
  }
}

template <typename T>
__global__ __launch_bounds__(256) void lru_conv_kernel(SeqView sv, LruArgs A,
                                                       T* __restrict__ u) {
  const int c = blockIdx.x * 256 + threadIdx.x;
  if (c >= A.C) return;
  const int r1 = min((int)(blockIdx.y + 1) * RC, sv.n);
  for (int row = blockIdx.y * RC; row < r1; ++row) {
    const int s = sv.seq[row], slot = sv.slots[s], row0 = sv.cu[s];
    stf(u + (u64)row * A.C + c,
        conv_at<T>(A, row, row0, sv.lens[slot] + row - row0, slot, c));
  }
}

// A workgroup = 64 tokens of one sequence x 64 channels of one block.
// ab [n, C] {decay, state} from the tile's start; ends [tiles, C] of a tile
__global__ __launch_bounds__(256) void lru_gates_mfma(
    SeqView sv, LruArgs A, const bf16_t* __restrict__ u,
    const i32* __restrict__ tile0, float2* __restrict__ ab,
    float2* __restrict__ ends) {
  constexpr int ROW = KC * 2 + 16;
  __shared__ __attribute__((aligned(16))) char us[TM * ROW];
  const int s = blockIdx.z, q0 = blockIdx.x * TM;
  const int row0 = sv.cu[s], cnt = sv.cu[s + 1] - row0;
  if (q0 >= cnt) return;
  const int ntile = (A.n + 63) / 64;
  const int blk = blockIdx.y / ntile;
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  const int l15 = lane & 15, l4 = lane >> 4;
  const int ch = blockIdx.y % ntile * 64 + wave * 16 + l15;   // in the block
  const bool on = ch < A.n;
  const bf16_t* wr = (const bf16_t*)A.gw +
                     ((u64)blk * 2 * A.n + (on ? ch : 0)) * A.n;
  const bf16_t* wi = wr + (u64)A.n * A.n;
  const s16x8 z8 = {0, 0, 0, 0, 0, 0, 0, 0};
  f32x4 ar[4] = {}, ai[4] = {};
  for (int k0 = 0; k0 < A.n; k0 += KC) {
    const int kn = min(KC, A.n - k0), kp = (kn + 31) / 32 * 32;
    __syncthreads();
    for (int id = tid; id < TM * (kp / 8); id += 256) {
      const int r = id / (kp / 8), e = (id % (kp / 8)) * 8;
      u32x4 d = {0, 0, 0, 0};
      if (e < kn && q0 + r < cnt)
        d = *(const u32x4*)(u + (u64)(row0 + q0 + r) * A.C + blk * A.n + k0 + e);
      *(u32x4*)(us + r * ROW + e * 2) = d;
    }
    __syncthreads();
    constexpr int U = 4;         // steps loaded ahead of their products
    for (int k = 0; k < kp; k += U * 32) {
      s16x8 br[U], bi[U];
#pragma unroll
      for (int i = 0; i < U; ++i) {
        const int kk = k + i * 32 + l4 * 8;
        br[i] = kk < kn ? *(const s16x8*)(wr + k0 + kk) : z8;
        bi[i] = kk < kn ? *(const s16x8*)(wi + k0 + kk) : z8;
      }
#pragma unroll
      for (int i = 0; i < U; ++i) {
        if (k + i * 32 >= kp) break;
        const int kk = k + i * 32 + l4 * 8;
#pragma unroll
        for (int mt = 0; mt < 4; ++mt) {
          const s16x8 a = *(const s16x8*)(us + (mt * 16 + l15) * ROW + kk * 2);
          ar[mt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, br[i], ar[mt],
                                                           0, 0, 0);
          ai[mt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, bi[i], ai[mt],
                                                           0, 0, 0);
        }
      }
    }
  }
  const int c = blk * A.n + (on ? ch : 0);
  const float csp = A.c * softplus_f(A.lam[c]);
  const float rb = A.gb[(u64)blk * 2 * A.n + (on ? ch : 0)];
  const float ib = A.gb[((u64)blk * 2 + 1) * A.n + (on ? ch : 0)];
  float ra = 1.f, rz = 0.f;      // up to this 16-token group
#pragma unroll
  for (int mt = 0; mt < 4; ++mt) {
    float a[4], z[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int row = q0 + mt * 16 + l4 * 4 + r;
      a[r] = 1.f;
      z[r] = 0.f;
      if (row < cnt)
        lru_pair<true>(ar[mt][r] + rb, ai[mt][r] + ib,
                       ldf(u + (u64)(row0 + row) * A.C + c), csp, a[r], z[r]);
      if (r) {
        z[r] = fmaf(a[r], z[r - 1], z[r]);
        a[r] *= a[r - 1];
      }
    }
    float pa = ra, pz = rz;      // up to this lane's four tokens
#pragma unroll
    for (int g = 0; g < 4; ++g) {
      const float ta = __shfl(a[3], l15 + 16 * g, 64);
      const float tz = __shfl(z[3], l15 + 16 * g, 64);
      if (g < l4) {
        pz = fmaf(ta, pz, tz);
        pa *= ta;
      }
      rz = fmaf(ta, rz, tz);
      ra *= ta;
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int row = q0 + mt * 16 + l4 * 4 + r;
      if (on && row < cnt)
        ab[(u64)(row0 + row) * A.C + c] =
            make_float2(a[r] * pa, fmaf(a[r], pz, z[r]));
    }
  }
  if (on && l4 == 0)
    ends[(u64)(tile0[s] + blockIdx.x) * A.C + c] = make_float2(ra, rz);
}

// the last inputs of the convolution go into the ring (one thread a channel
// of a sequence)
template <typename T>
__device__ __forceinline__ void keep_inputs(const SeqView& sv,
                                            const LruArgs& A, int s, int slot,
                                            int c) {
  const int row0 = sv.cu[s], n = sv.cu[s + 1] - row0, len0 = sv.lens[slot];
  for (int i = max(0, n - A.taps); i < n; ++i)
    A.ring[((u64)slot * A.taps + (len0 + i) % A.taps) * A.C + c] =
        ldf((const T*)A.x + (u64)(row0 + i) * A.ld + c) + A.xb[c];
}

// ends[tile].x becomes the state at the tile's start
__global__ __launch_bounds__(64) void lru_carry_kernel(
    SeqView sv, LruArgs A, const i32* __restrict__ tile0,
    float2* __restrict__ ends) {
  const int c = blockIdx.x * 64 + threadIdx.x, s = blockIdx.y;
  if (c >= A.C) return;
  const int slot = sv.slots[s];
  const int tiles = (sv.cu[s + 1] - sv.cu[s] + TM - 1) / TM;
  float S = sv.lens[slot] == 0 ? 0.f : A.S[(u64)slot * A.C + c];
  float2* e = ends + (u64)tile0[s] * A.C + c;
  constexpr int U = 16;
  for (int t0 = 0; t0 < tiles; t0 += U) {
    float2 v[U];
#pragma unroll
    for (int i = 0; i < U; ++i)
      v[i] = t0 + i < tiles ? e[(u64)(t0 + i) * A.C] : make_float2(1.f, 0.f);
#pragma unroll
    for (int i = 0; i < U; ++i) {
      if (t0 + i < tiles) e[(u64)(t0 + i) * A.C].x = S;
      S = fmaf(v[i].x, S, v[i].y);
    }
  }
  A.S[(u64)slot * A.C + c] = S;
  keep_inputs<bf16_t>(sv, A, s, slot, c);
}

template <int VEC>
__global__ __launch_bounds__(256) void lru_apply_kernel(
    SeqView sv, LruArgs A, const i32* __restrict__ tile0,
    const float2* __restrict__ ab, const float2* __restrict__ ends) {
  const int c = (blockIdx.x * 256 + threadIdx.x) * VEC;
  if (c >= A.C) return;
  float yb[VEC];
  ldv<float, VEC>(A.yb + c, yb);
  const int r1 = min((int)(blockIdx.y + 1) * RC, sv.n);
  for (int row = blockIdx.y * RC; row < r1; ++row) {
    const int s = sv.seq[row];
    const float2* e =
        ends + (u64)(tile0[s] + (row - sv.cu[s]) / TM) * A.C + c;
    const float2* p = ab + (u64)row * A.C + c;
    float y[VEC];
    ldv<bf16_t, VEC>((const bf16_t*)A.y + (u64)row * A.ld + c, y);
    float2 q[VEC];
    float st[VEC];
#pragma unroll
    for (int i = 0; i < VEC; ++i) {
      q[i] = p[i];
      st[i] = e[i].x;
    }
#pragma unroll
    for (int i = 0; i < VEC; ++i)
      y[i] = A.gain * fmaf(q[i].x, st[i], q[i].y) *
             gelu_tanh_f<true>(y[i] + yb[i]);
    stv<bf16_t, VEC>((bf16_t*)A.out + (u64)row * A.ldo + c, y);
  }
}

// One token of up to 16 sequences x CT * 16 channels of a block: a wave has
// 16 channels and a quarter of the gates' inner dimension.  TAPS 0: any
// number of them.
constexpr int MAX_TAPS = 16;

template <int CT, int TAPS>
__global__ __launch_bounds__(CT * 256) void lru_step_mfma(SeqView sv,
                                                          LruArgs A) {
  constexpr int ROW = SKC * 2 + 16, KW = 4, NC = CT * 16, TPB = CT * 256;
  const int taps = TAPS ? TAPS : A.taps;
  __shared__ __attribute__((aligned(16))) char us[16 * ROW];
  __shared__ float red[KW][2][16][NC + 1];
  __shared__ int back[MAX_TAPS][16];     // ring row of an earlier input, or -1
  const int b0 = blockIdx.z * 16, nb = min(16, sv.b - b0);
  const int blk = blockIdx.y, n0 = blockIdx.x * NC;
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  const int l15 = lane & 15, l4 = lane >> 4;
  const int ct = wave % CT, kw = wave / CT;
  const int ch = min(n0 + ct * 16 + l15, A.n - 1);
  const bf16_t* wr = (const bf16_t*)A.gw + ((u64)blk * 2 * A.n + ch) * A.n;
  const bf16_t* wi = wr + (u64)A.n * A.n;
  const s16x8 z8 = {0, 0, 0, 0, 0, 0, 0, 0};
  for (int id = tid; id < 16 * taps; id += TPB) {
    const int i = id & 15, j = id >> 4;
    if (i < nb) {
      const int slot = sv.slots[b0 + i], p = sv.lens[slot] - j;
      back[j][i] = p >= 0 ? slot * taps + p % taps : -1;
    }
  }
  f32x4 ar = {}, ai = {};
  for (int k0 = 0; k0 < A.n; k0 += SKC) {
    const int kn = min(SKC, A.n - k0), kp = (kn + 31) / 32 * 32;
    __syncthreads();
    for (int id = tid; id < nb * (kp / 4); id += TPB) {
      const int i = id / (kp / 4), k = (id % (kp / 4)) * 4;
      float v[4] = {};
      if (k < kn) {
        const int c = blk * A.n + k0 + k;
        float t[4], w[4];
        ldf4(A.cb + c, v);
#pragma unroll
        for (int j = taps - 1; j > 0; --j) {
          const int row = back[j][i];
          ldf4(A.ring + (u64)max(row, 0) * A.C + c, t);
          ldf4(A.cw + (u64)(taps - 1 - j) * A.C + c, w);
#pragma unroll
          for (int e = 0; e < 4; ++e)
            v[e] = row < 0 ? v[e] : fmaf(w[e], t[e], v[e]);
        }
        float xb[4];
        load_x4<bf16_t>(A, b0 + i, c, t);
        ldf4(A.xb + c, xb);
        ldf4(A.cw + (u64)(taps - 1) * A.C + c, w);
#pragma unroll
        for (int e = 0; e < 4; ++e) v[e] = fmaf(w[e], t[e] + xb[e], v[e]);
      }
      stf4((bf16_t*)(us + i * ROW) + k, v);
    }
    __syncthreads();
    constexpr int U = 2;
    for (int k = kw * 32; k < kp; k += U * KW * 32) {
      s16x8 br[U], bi[U];
#pragma unroll
      for (int i = 0; i < U; ++i) {
        const int kk = k + i * KW * 32 + l4 * 8;
        br[i] = kk < kn ? *(const s16x8*)(wr + k0 + kk) : z8;
        bi[i] = kk < kn ? *(const s16x8*)(wi + k0 + kk) : z8;
      }
#pragma unroll
      for (int i = 0; i < U; ++i) {
        const int kk = k + i * KW * 32 + l4 * 8;
        const s16x8 a = l15 < nb && kk < kp
                            ? *(const s16x8*)(us + l15 * ROW + kk * 2)
                            : z8;
        ar = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, br[i], ar, 0, 0, 0);
        ai = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, bi[i], ai, 0, 0, 0);
      }
    }
  }
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    red[kw][0][l4 * 4 + r][ct * 16 + l15] = ar[r];
    red[kw][1][l4 * 4 + r][ct * 16 + l15] = ai[r];
  }
  __syncthreads();
  for (int id = tid; id < nb * NC; id += TPB) {
    const int i = id / NC, j = id % NC;
    if (n0 + j >= A.n) continue;
    float r = A.gb[(u64)blk * 2 * A.n + n0 + j];
    float g = A.gb[((u64)blk * 2 + 1) * A.n + n0 + j];
#pragma unroll
    for (int w = 0; w < KW; ++w) {
      r += red[w][0][i][j];
      g += red[w][1][i][j];
    }
    const int row = b0 + i, slot = sv.slots[row], pos = sv.lens[slot];
    const int c = blk * A.n + n0 + j;
    const float x = ldf((const bf16_t*)A.x + (u64)row * A.ld + c) + A.xb[c];
    float u = A.cb[c];
#pragma unroll
    for (int t = taps - 1; t > 0; --t) {
      const int br = back[t][i];
      const float v = fmaf(A.cw[(u64)(taps - 1 - t) * A.C + c],
                           A.ring[(u64)max(br, 0) * A.C + c], u);
      u = br < 0 ? u : v;
    }
    u = fmaf(A.cw[(u64)(taps - 1) * A.C + c], x, u);
    float a, z;
    lru_pair<true>(r, g, round_to(u, (const bf16_t*)nullptr),
                   A.c * softplus_f(A.lam[c]), a, z);
    float* sp = A.S + (u64)slot * A.C + c;
    const float S = fmaf(a, pos == 0 ? 0.f : *sp, z);
    *sp = S;
    A.ring[(u64)back[0][i] * A.C + c] = x;     // no one reads this row
    const float y = ldf((const bf16_t*)A.y + (u64)row * A.ld + c) + A.yb[c];
    stf((bf16_t*)A.out + (u64)row * A.ldo + c,
        A.gain * S * gelu_tanh_f<true>(y));
  }
}

// any size: a workgroup = one row of one block, a wave a channel at a time
template <typename T>
__global__ __launch_bounds__(256) void lru_gates_any(
    SeqView sv, LruArgs A, const T* __restrict__ u, float2* __restrict__ ab) {
  extern __shared__ float ub[];      // [n]
  const int row = blockIdx.x, blk = blockIdx.y;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  for (int k = threadIdx.x; k < A.n; k += 256)
    ub[k] = ldf(u + (u64)row * A.C + blk * A.n + k);
  __syncthreads();
  for (int j = wave; j < A.n; j += 4) {
    const T* wr = (const T*)A.gw + ((u64)blk * 2 * A.n + j) * A.n;
    const T* wi = wr + (u64)A.n * A.n;
    float r = 0.f, g = 0.f;
    for (int k = lane; k < A.n; k += 64) {
      r = fmaf(ldf(wr + k), ub[k], r);
      g = fmaf(ldf(wi + k), ub[k], g);
    }
    r = wave_reduce_sum(r) + A.gb[(u64)blk * 2 * A.n + j];
    g = wave_reduce_sum(g) + A.gb[((u64)blk * 2 + 1) * A.n + j];
    if (lane == 0) {
      const int c = blk * A.n + j;
      float a, z;
      lru_pair<false>(r, g, ub[j], A.c * softplus_f(A.lam[c]), a, z);
      ab[(u64)row * A.C + c] = make_float2(a, z);
    }
  }
}

// token by token, a thread per channel of a sequence
template <typename T>
__global__ __launch_bounds__(64) void lru_scan_kernel(
    SeqView sv, LruArgs A, const float2* __restrict__ ab) {
  const int c = blockIdx.x * 64 + threadIdx.x, s = blockIdx.y;
  if (c >= A.C) return;
  const int slot = sv.slots[s];
  float S = sv.lens[slot] == 0 ? 0.f : A.S[(u64)slot * A.C + c];
#pragma unroll 4
  for (int row = sv.cu[s]; row < sv.cu[s + 1]; ++row) {
    const float2 p = ab[(u64)row * A.C + c];
    S = fmaf(p.x, S, p.y);
    const float y = ldf((const T*)A.y + (u64)row * A.ld + c) + A.yb[c];
    stf((T*)A.out + (u64)row * A.ldo + c, A.gain * S * gelu_tanh_f<false>(y));
  }
  A.S[(u64)slot * A.C + c] = S;
  keep_inputs<T>(sv, A, s, slot, c);
}

LruArgs args(const void* x, const void* y, long ld, const void* xb,
             const void* yb, const void* cw, const void* cb, const void* gw,
             const void* gb, const void* lam, void* ring, void* S, void* out,
             long ldo, int C, int blocks, int taps, float c, float gain) {
  return LruArgs{x, y, (u64)ld, (const float*)xb, (const float*)yb,
                 (const float*)cw, (const float*)cb, (const float*)gb,
                 (const float*)lam, gw, (float*)ring, (float*)S, out,
                 (u64)ldo, C, blocks, C / blocks, taps, c, gain,
                 ld % 4 == 0 && ((u64)x & 15) == 0};
}

}  // namespace

bool lfmq_lru_mfma_ok(const void* gw, int n, int taps) {
  return n % 8 == 0 && taps <= MAX_TAPS && ((u64)gw & 15) == 0;
}

// prompts: u [n, C], ab [n, C, 2], ends [tiles, C, 2] scratch; tile0 [b]
// first 64-token tile of a sequence.  single: one token per sequence, no
// scratch.  mfma false: the any-size kernels (no tiles).
hipError_t lfmq_gated_lru(const SeqView& sv, const void* x, const void* y,
                          long ld, const void* xb, const void* yb,
                          const void* cw, const void* cb, const void* gw,
                          const void* gb, const void* lam, void* ring,
                          void* S, void* out, long ldo, int C, int blocks,
                          int taps, float c, float gain, void* u, void* ab,
                          void* ends, const void* tile0, int max_count,
                          bool single, bool mfma, bool f32,
                          hipStream_t stream) {
  const LruArgs A = args(x, y, ld, xb, yb, cw, cb, gw, gb, lam, ring, S, out,
                         ldo, C, blocks, taps, c, gain);
  if (mfma && single) {
    // wide tiles compute each convolution output less often, narrow ones
    // spread few sequences over the chip
#define STEP(CT)                                                             \
  do {                                                                       \
    const dim3 grid((A.n + CT * 16 - 1) / (CT * 16), blocks,                 \
                    (sv.b + 15) / 16);                                       \
    if (taps == 4)                                                           \
      hipLaunchKernelGGL((lru_step_mfma<CT, 4>), grid, dim3(CT * 256), 0,    \
                         stream, sv, A);                                     \
    else                                                                     \
      hipLaunchKernelGGL((lru_step_mfma<CT, 0>), grid, dim3(CT * 256), 0,    \
                         stream, sv, A);                                     \
  } while (0)
    if (sv.b >= 16) STEP(4); else STEP(1);
#undef STEP
    return hipGetLastError();
  }
  const bool c4 = taps == 4 && C % 4 == 0;
  const int per = c4 ? 1024 : 256;
  const dim3 conv_grid((C + per - 1) / per, (sv.n + RC - 1) / RC);
  if (conv_grid.y > 65535) return hipErrorInvalidValue;
#define CONV(T)                                                              \
  do {                                                                       \
    if (c4)                                                                  \
      hipLaunchKernelGGL(lru_conv4_kernel<T>, conv_grid, dim3(256), 0,       \
                         stream, sv, A, (T*)u);                              \
    else                                                                     \
      hipLaunchKernelGGL(lru_conv_kernel<T>, conv_grid, dim3(256), 0,        \
                         stream, sv, A, (T*)u);                              \
  } while (0)
  if (f32) CONV(float); else CONV(bf16_t);
#undef CONV
  const dim3 chan_grid((C + 63) / 64, sv.b);
  if (mfma) {
    hipLaunchKernelGGL(lru_gates_mfma,
                       dim3((max_count + TM - 1) / TM,
                            blocks * ((A.n + 63) / 64), sv.b),
                       dim3(256), 0, stream, sv, A, (const bf16_t*)u,
                       (const i32*)tile0, (float2*)ab, (float2*)ends);
    hipLaunchKernelGGL(lru_carry_kernel, chan_grid, dim3(64), 0, stream, sv,
                       A, (const i32*)tile0, (float2*)ends);
    const bool v4 = C % 4 == 0 && ld % 4 == 0 && ldo % 4 == 0 &&
                    (((u64)y | (u64)out) & 7) == 0 && ((u64)yb & 15) == 0;
    const int ap = v4 ? 1024 : 256;
    const dim3 ag((C + ap - 1) / ap, (sv.n + RC - 1) / RC);
    if (v4)
      hipLaunchKernelGGL(lru_apply_kernel<4>, ag, dim3(256), 0, stream, sv, A,
                         (const i32*)tile0, (const float2*)ab,
                         (const float2*)ends);
    else
      hipLaunchKernelGGL(lru_apply_kernel<1>, ag, dim3(256), 0, stream, sv, A,
                         (const i32*)tile0, (const float2*)ab,
                         (const float2*)ends);
    return hipGetLastError();
  }
  const size_t lds = (size_t)A.n * sizeof(float);
  if (lds > 64 * 1024) return hipErrorInvalidValue;
  const dim3 gate_grid(sv.n, blocks);
  if (f32) {
    hipLaunchKernelGGL(lru_gates_any<float>, gate_grid, dim3(256), lds,
                       stream, sv, A, (const float*)u, (float2*)ab);
    hipLaunchKernelGGL(lru_scan_kernel<float>, chan_grid, dim3(64), 0, stream,
                       sv, A, (const float2*)ab);
  } else {
    hipLaunchKernelGGL(lru_gates_any<bf16_t>, gate_grid, dim3(256), lds,
                       stream, sv, A, (const bf16_t*)u, (float2*)ab);
    hipLaunchKernelGGL(lru_scan_kernel<bf16_t>, chan_grid, dim3(64), 0,
                       stream, sv, A, (const float2*)ab);
  }
  return hipGetLastError();
}
