// Chunk-parallel matrix-memory LSTM on the matrix cores, for 16-bit
// prompts (mlstm.hip states the recurrence and runs it token by token).
//
// A sequence is cut into chunks of L tokens.  With F the running sum of
// the log forget gates inside a chunk, m_t the running maximum and m_c its
// value at the chunk's start, every weight is an exponential of something
// <= 0:
//   intra   P_ts = q_t.k_s exp((F_t - m_t) + (i_s - F_s))        s <= t
//   inter   c_t  = exp(F_t + m_c - m_t)
//   o_t = (sum_s P_ts v_s + c_t S_c^T q_t) /
//         (max(|sum_s P_ts + c_t n_c.q_t|, exp(-m_t)) + 1e-6)
//   S_c+1 = exp(F_L + m_c - m_L) S_c + sum_s exp(F_L - F_s + i_s - m_L) k_s v_s^T
//
// Three kernels:
//   gates   scan of (F, m) per head: (+, max) composition over 1024
//           tokens at a time
//   states  S and n at every chunk start.  A workgroup owns a 64 x 64 tile
//           of S in accumulators and walks the sequence, the next tokens'
//           rows in flight while it multiplies
//   output  64 queries x all of vdim per workgroup, 8 waves splitting
//           vdim; head norm, weight and output gate in the epilogue
//
// Operands that must keep 32 bits (S, the decayed keys, P) go through the
// 16-bit matrix cores as a sum of two bf16 parts; q, k and v are bf16
// already.  S lives transposed [v][d] between the kernels, so that its
// fragments are contiguous 16-byte loads.
#include "seq_common.h"

#include "mlstm_gate.h"

namespace {

__device__ __forceinline__ u32 swz(u32 row) { return (row ^ (row >> 3)) & 7; }

// ---- gates ---------------------------------------------------------------
constexpr int GT = 1024, GW = GT / 64;

__global__ __launch_bounds__(GT) void mlstm_gate_scan_kernel(
    const float* __restrict__ gates, SeqView sv, const i32* __restrict__ turn,
    float* __restrict__ nm, float* __restrict__ gF, float* __restrict__ gI,
    float* __restrict__ gM, int heads, int dim, float cap, int waves_per_chunk) {
  const int h = blockIdx.x, s = blockIdx.y;
  const int n0 = sv.cu[s], n1 = sv.cu[s + 1];
  if (n1 <= n0) return;
  const int slot = sv.slots[s], cur = turn[slot] & 1;
  const bool fresh = sv.lens[slot] == 0;
  const u64 st = (u64)heads * (dim + 1), at = (u64)h * (dim + 1) + dim;
  float m = fresh ? 0.f : nm[((u64)slot * 2 + cur) * st + at];
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  __shared__ float wF[GW], wM[GW];
  float ri = 0.f, rf = 0.f;                  // raw gates, one block ahead
  auto fetch = [&](int row) {
    if (row < n1) {
      const float* g = gates + (u64)row * 2 * heads + h;
      ri = g[0];
      rf = g[heads];
    }
  };
  fetch(n0 + threadIdx.x);
  for (int b0 = n0; b0 < n1; b0 += GT) {
    const int row = b0 + threadIdx.x;
    const bool live = row < n1;
    const float gi = live ? mlstm_input_gate(ri, cap) : -INFINITY;
    float F = live ? mlstm_forget_gate(rf, cap) : 0.f;
    fetch(row + GT);
    float M = gi;
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const float Fp = __shfl_up(F, o, 64), Mp = __shfl_up(M, o, 64);
      if (lane >= o) {
        M = fmaxf(Mp + F, M);
        F += Fp;
      }
    }
    if (lane == 63) {
      wF[wave] = F;
      wM[wave] = M;
    }
    __syncthreads();
    float mc = m, Floc = F;
    for (int w = 0; w < GW; ++w) {
      if (w < wave) {
        mc = fmaxf(wF[w] + mc, wM[w]);
        if (w >= wave - wave % waves_per_chunk) Floc += wF[w];
      }
      m = fmaxf(wF[w] + m, wM[w]);
    }
    if (live) {
      const u64 o = (u64)h * sv.n + row;
      gF[o] = Floc;
      gI[o] = gi;
      gM[o] = fmaxf(F + mc, M);
    }
    __syncthreads();
  }
  if (threadIdx.x == 0) nm[((u64)slot * 2 + (cur ^ 1)) * st + at] = m;
}

struct CArgs {
  const bf16_t* qkv;       // rows [q (H dim) | k (H dim) | v (H vdim) | g]
  u64 ld;
  const float *gF, *gI, *gM;
  const i32 *turn, *chunk_base;
  float *S, *nm;
  unsigned short* ws;      // [chunks, H, 2 (hi, lo), VP, DP]
  float* nws;              // [chunks, H, DP]
  const float* norm_w;
  bf16_t* out;             // [N, H vdim]
  int heads, dim, vdim, L, DP, VP;
  float eps;
};

// ---- states ----------------------------------------------------------------
struct Rows2 {             // two tokens x 8 columns, and their gates
  u32x4 ka, kb, va, vb;
  float fa, fb, ia, ib;
};

__device__ __forceinline__ Rows2 load_rows(const CArgs& A, const u64 ho,
                                           int h, int ra, int n1, int d,
                                           int v) {
  Rows2 r;
  const u32x4 z = {0, 0, 0, 0};
  const bool oa = ra < n1, ob = ra + 1 < n1;
  const bf16_t* p = A.qkv + (u64)ra * A.ld;
  const u64 ko = (u64)(A.heads + h) * A.dim + d;
  const u64 vo = (u64)2 * A.heads * A.dim + (u64)h * A.vdim + v;
  const bool dk = d < A.dim, dv = v < A.vdim;
  r.ka = (oa && dk) ? *(const u32x4*)(p + ko) : z;
  r.kb = (ob && dk) ? *(const u32x4*)(p + A.ld + ko) : z;
  r.va = (oa && dv) ? *(const u32x4*)(p + vo) : z;
  r.vb = (ob && dv) ? *(const u32x4*)(p + A.ld + vo) : z;
  r.fa = oa ? A.gF[ho + ra] : 0.f;
  r.fb = ob ? A.gF[ho + ra + 1] : 0.f;
  r.ia = oa ? A.gI[ho + ra] : -INFINITY;     // weight 0
  r.ib = ob ? A.gI[ho + ra + 1] : -INFINITY;
  return r;
}

__global__ __launch_bounds__(256) void mlstm_states_kernel(SeqView sv,
                                                           CArgs A) {
  __shared__ __attribute__((aligned(16))) char kh[64 * 128], kl[64 * 128],
      vt[64 * 128];
  const int h = blockIdx.y, s = blockIdx.z;
  const int n0 = sv.cu[s], n1 = sv.cu[s + 1];
  if (n1 <= n0) return;
  const int slot = sv.slots[s], cur = A.turn[slot] & 1;
  const bool fresh = sv.lens[slot] == 0;
  const int dtiles = A.DP / 64;
  const int d0 = (blockIdx.x % dtiles) * 64, v0 = (blockIdx.x / dtiles) * 64;
  const bool has_n = v0 == 0;
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  const int l15 = lane & 15, l4 = lane >> 4;
  float* S = A.S + ((u64)slot * A.heads + h) * A.dim * A.vdim;
  const u64 nms = (u64)A.heads * (A.dim + 1);
  const float* nm_in = A.nm + ((u64)slot * 2 + cur) * nms +
                       (u64)h * (A.dim + 1);
  float* nm_out = A.nm + ((u64)slot * 2 + (cur ^ 1)) * nms +
                  (u64)h * (A.dim + 1);
  const u64 ho = (u64)h * sv.n;

  const int dr = d0 + wave * 16 + l4 * 4;   // this lane's 4 rows of S
  f32x4 acc[4];
#pragma unroll
  for (int nt = 0; nt < 4; ++nt) {
    const int v = v0 + nt * 16 + l15;
#pragma unroll
    for (int r = 0; r < 4; ++r)
      acc[nt][r] = (!fresh && dr + r < A.dim && v < A.vdim)
                       ? S[(u64)(dr + r) * A.vdim + v] : 0.f;
  }
  const int nd = d0 + (tid >> 2);           // n: 4 threads an element
  float nv = (has_n && !fresh && nd < A.dim) ? nm_in[nd] : 0.f;
  float mst = fresh ? 0.f : nm_in[A.dim];

  // staging role: token pair tp, 8 columns cg
  const int cg = tid & 7, tp = tid >> 3;
  const int per = A.L / 64;
  const int nsb = (n1 - n0 + 63) / 64;
  Rows2 nx = load_rows(A, ho, h, n0 + 2 * tp, n1, d0 + cg * 8, v0 + cg * 8);
  int rl = min(n1, n0 + A.L) - 1;
  float FLn = A.gF[ho + rl], mLn = A.gM[ho + rl], FL = 0.f, mL = 0.f;
  for (int sb = 0; sb < nsb; ++sb) {
    const Rows2 c = nx;
    if (sb % per == 0) {
      // chunk start: hand S and n to the output kernel, then decay them
      FL = FLn;
      mL = mLn;
      if (sb > 0 || !fresh) {
        const u64 cid = A.chunk_base[s] + sb / per;
        unsigned short* w = A.ws + (cid * A.heads + h) * 2 * A.VP * A.DP;
#pragma unroll
        for (int nt = 0; nt < 4; ++nt) {
          const u64 o = (u64)(v0 + nt * 16 + l15) * A.DP + dr;
          unsigned short hi[4], lo[4];
#pragma unroll
          for (int r = 0; r < 4; ++r) split_bf16(acc[nt][r], hi[r], lo[r]);
          *(u32x2*)(w + o) = u32x2{hi[0] | ((u32)hi[1] << 16),
                                   hi[2] | ((u32)hi[3] << 16)};
          *(u32x2*)(w + (u64)A.VP * A.DP + o) =
              u32x2{lo[0] | ((u32)lo[1] << 16), lo[2] | ((u32)lo[3] << 16)};
        }
        if (has_n && (tid & 3) == 0)
          A.nws[(cid * A.heads + h) * A.DP + nd] = nv;
      }
      const float a = expf(FL + mst - mL);
      mst = mL;
#pragma unroll
      for (int nt = 0; nt < 4; ++nt)
#pragma unroll
        for (int r = 0; r < 4; ++r) acc[nt][r] *= a;
      nv *= a;
    }
    const float wa = expf(FL - c.fa + c.ia - mL);
    const float wb = expf(FL - c.fb + c.ib - mL);
    __syncthreads();          // the last tile's fragments are read
    {
      const u32 blk = tp >> 2, off = (tp & 3) * 4;
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        const u32 row = cg * 8 + e;
        const u32 o = row * 128 + ((blk ^ swz(row)) << 4) + off;
        const u32 sh = (e & 1) * 16;
        unsigned short ha, la, hb, lb;
        split_bf16(wa * bf16_bits_to_f32((c.ka[e >> 1] >> sh) & 0xFFFFu), ha,
                   la);
        split_bf16(wb * bf16_bits_to_f32((c.kb[e >> 1] >> sh) & 0xFFFFu), hb,
                   lb);
        *(u32*)(kh + o) = ha | ((u32)hb << 16);
        *(u32*)(kl + o) = la | ((u32)lb << 16);
        *(u32*)(vt + o) = ((c.va[e >> 1] >> sh) & 0xFFFFu) |
                          (((c.vb[e >> 1] >> sh) & 0xFFFFu) << 16);
      }
    }
    if (sb + 1 < nsb) {
      nx = load_rows(A, ho, h, n0 + (sb + 1) * 64 + 2 * tp, n1, d0 + cg * 8,
                     v0 + cg * 8);
      if ((sb + 1) % per == 0) {
        rl = min(n1, n0 + (sb + 1) * 64 + A.L) - 1;
        FLn = A.gF[ho + rl];
        mLn = A.gM[ho + rl];
      }
    }
    __syncthreads();
#pragma unroll
    for (int ks = 0; ks < 2; ++ks) {
      const u32 ar = wave * 16 + l15, blk = ks * 4 + l4;
      const u32 ao = ar * 128 + ((blk ^ swz(ar)) << 4);
      const s16x8 ah = *(const s16x8*)(kh + ao);
      const s16x8 al = *(const s16x8*)(kl + ao);
#pragma unroll
      for (int nt = 0; nt < 4; ++nt) {
        const u32 br = nt * 16 + l15;
        const s16x8 b =
            *(const s16x8*)(vt + br * 128 + ((blk ^ swz(br)) << 4));
        acc[nt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ah, b, acc[nt], 0,
                                                          0, 0);
        acc[nt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(al, b, acc[nt], 0,
                                                          0, 0);
      }
    }
    if (has_n) {
      const u32 row = tid >> 2;
      float t = 0.f;
#pragma unroll
      for (int j = 0; j < 2; ++j) {
        const u32 blk = (tid & 3) * 2 + j;
        const u32 o = row * 128 + ((blk ^ swz(row)) << 4);
        const u32x4 x = *(const u32x4*)(kh + o), y = *(const u32x4*)(kl + o);
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          float p, q;
          bf16x2_to_f32(x[e], p, q);
          t += p + q;
          bf16x2_to_f32(y[e], p, q);
          t += p + q;
        }
      }
      t += __shfl_xor(t, 1, 64);
      t += __shfl_xor(t, 2, 64);
      nv += t;
    }
  }
#pragma unroll
  for (int nt = 0; nt < 4; ++nt) {
    const int v = v0 + nt * 16 + l15;
#pragma unroll
    for (int r = 0; r < 4; ++r)
      if (dr + r < A.dim && v < A.vdim)
        S[(u64)(dr + r) * A.vdim + v] = acc[nt][r];
  }
  if (has_n && (tid & 3) == 0 && nd < A.dim) nm_out[nd] = nv;
}

// ---- output ------------------------------------------------------------------
template <int KS, int NTW>
constexpr size_t out_lds() {
  constexpr size_t krow = KS * 64 + 16, vrows = 128 * NTW;
  constexpr size_t x = 64 * krow > vrows * 128 ? 64 * krow : vrows * 128;
  return 64 * krow + x + 2 * 64 * 144 + (5 * 64 + 2 * 64 + 8 * 64) * 4;
}

template <int KS, int NTW>
__global__ __launch_bounds__(512) void mlstm_out_kernel(SeqView sv, CArgs A) {
  constexpr int DQ = KS * 32, KROW = DQ * 2 + 16, VR = 128 * NTW;
  constexpr int XB = 64 * KROW > VR * 128 ? 64 * KROW : VR * 128;
  constexpr int PROW = 144;
  extern __shared__ __attribute__((aligned(16))) char smem[];
  char* ldsQ = smem;
  char* ldsX = ldsQ + 64 * KROW;       // keys, then transposed values
  char* ldsPh = ldsX + XB;
  char* ldsPl = ldsPh + 64 * PROW;
  float* At = (float*)(ldsPl + 64 * PROW);   // F_t - m_t
  float* Ct = At + 64;                       // c_t / sqrt(dim)
  float* Mt = Ct + 64;
  float* Bs = Mt + 64;                       // i_s - F_s
  float* sc = Bs + 64;
  float* denp = sc + 64;                     // [2][64]
  float* red = denp + 128;                   // [8][64]

  const int s = blockIdx.z, h = blockIdx.y, q0 = blockIdx.x * 64;
  const int n0 = sv.cu[s], cnt = sv.cu[s + 1] - n0;
  if (q0 >= cnt) return;
  const int slot = sv.slots[s];
  const bool fresh = sv.lens[slot] == 0;
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  const int l15 = lane & 15, l4 = lane >> 4;
  const int c = q0 / A.L, cr0 = c * A.L;     // chunk, its first local row
  const bool inter = c > 0 || !fresh;
  const u64 cid = A.chunk_base[s] + c;
  const u64 ho = (u64)h * sv.n + n0;
  const float qscale = 1.f / sqrtf((float)A.dim);
  const bf16_t* rows = A.qkv + (u64)n0 * A.ld;
  const u64 koff = (u64)(A.heads + h) * A.dim;
  const u64 voff = (u64)2 * A.heads * A.dim + (u64)h * A.vdim;

  for (int i = tid; i < 64 * (DQ / 8); i += 512) {
    const int r = i / (DQ / 8), d = (i % (DQ / 8)) * 8;
    u32x4 x = {0, 0, 0, 0};
    if (q0 + r < cnt && d < A.dim)
      x = *(const u32x4*)(rows + (u64)(q0 + r) * A.ld + (u64)h * A.dim + d);
    *(u32x4*)(ldsQ + r * KROW + d * 2) = x;
  }
  if (tid < 64) {
    const bool ok = q0 + tid < cnt;
    const float F = ok ? A.gF[ho + q0 + tid] : 0.f;
    const float m = ok ? A.gM[ho + q0 + tid] : 0.f;
    float mc = 0.f;
    if (c > 0) mc = A.gM[ho + cr0 - 1];
    else if (!fresh)
      mc = A.nm[(((u64)slot * 2 + (A.turn[slot] & 1)) * A.heads + h) *
                    (A.dim + 1) + A.dim];
    At[tid] = F - m;
    Mt[tid] = m;
    Ct[tid] = ok && inter ? expf(F + mc - m) * qscale : 0.f;
    denp[tid] = 0.f;
    denp[64 + tid] = 0.f;
  }
  __syncthreads();

  f32x4 acc[4][NTW] = {};
  if (inter) {
    const unsigned short* w = A.ws + (cid * A.heads + h) * 2 * A.VP * A.DP;
    const u64 lo_off = (u64)A.VP * A.DP;
#pragma unroll 2
    for (int ks = 0; ks < KS; ++ks) {
      const int k = ks * 32 + l4 * 8;
      s16x8 bh[NTW], bl[NTW];
#pragma unroll
      for (int j = 0; j < NTW; ++j) {
        const int v = (wave * NTW + j) * 16 + l15;
        const s16x8 z = {0, 0, 0, 0, 0, 0, 0, 0};
        const bool ok = v < A.VP && k < A.DP;
        const unsigned short* p = w + (u64)v * A.DP + k;
        bh[j] = ok ? *(const s16x8*)p : z;
        bl[j] = ok ? *(const s16x8*)(p + lo_off) : z;
      }
#pragma unroll
      for (int mt = 0; mt < 4; ++mt) {
        const s16x8 a = *(const s16x8*)(ldsQ + (mt * 16 + l15) * KROW + k * 2);
#pragma unroll
        for (int j = 0; j < NTW; ++j) {
          acc[mt][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, bh[j],
                                                               acc[mt][j], 0,
                                                               0, 0);
          acc[mt][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, bl[j],
                                                               acc[mt][j], 0,
                                                               0, 0);
        }
      }
    }
#pragma unroll
    for (int mt = 0; mt < 4; ++mt)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const float cf = Ct[mt * 16 + l4 * 4 + r];
#pragma unroll
        for (int j = 0; j < NTW; ++j) acc[mt][j][r] *= cf;
      }
  }

  const int mt0 = wave & 3, nh = wave >> 2;   // this wave's score tiles
  for (int k0 = cr0; k0 <= q0; k0 += 64) {
    __syncthreads();                          // X and P are free
    for (int i = tid; i < 64 * (DQ / 8); i += 512) {
      const int r = i / (DQ / 8), d = (i % (DQ / 8)) * 8;
      u32x4 x = {0, 0, 0, 0};
      if (k0 + r < cnt && d < A.dim)
        x = *(const u32x4*)(rows + (u64)(k0 + r) * A.ld + koff + d);
      *(u32x4*)(ldsX + r * KROW + d * 2) = x;
    }
    if (tid < 64)
      Bs[tid] = k0 + tid < cnt ? A.gI[ho + k0 + tid] - A.gF[ho + k0 + tid]
                               : 0.f;
    __syncthreads();
    f32x4 p[2] = {};
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
      const int ko = (ks * 32 + l4 * 8) * 2;
      const s16x8 a = *(const s16x8*)(ldsQ + (mt0 * 16 + l15) * KROW + ko);
#pragma unroll
      for (int j = 0; j < 2; ++j) {
        const s16x8 b =
            *(const s16x8*)(ldsX + ((nh * 2 + j) * 16 + l15) * KROW + ko);
        p[j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, p[j], 0, 0, 0);
      }
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int t = mt0 * 16 + l4 * 4 + r;
      float sum = 0.f;
#pragma unroll
      for (int j = 0; j < 2; ++j) {
        const int key = (nh * 2 + j) * 16 + l15;
        const bool ok = k0 + key <= q0 + t && q0 + t < cnt;
        const float x = ok ? p[j][r] * qscale * expf(At[t] + Bs[key]) : 0.f;
        sum += x;
        unsigned short hi, lo;
        split_bf16(x, hi, lo);
        *(unsigned short*)(ldsPh + t * PROW + key * 2) = hi;
        *(unsigned short*)(ldsPl + t * PROW + key * 2) = lo;
      }
#pragma unroll
      for (int o = 8; o > 0; o >>= 1) sum += __shfl_xor(sum, o, 64);
      if (l15 == 0) denp[nh * 64 + t] += sum;
    }
    __syncthreads();                          // keys are read, P is whole
    for (int i = tid; i < 32 * (VR / 8); i += 512) {
      const int kp = i / (VR / 8), dg = i % (VR / 8);
      u32x4 a = {0, 0, 0, 0}, b = {0, 0, 0, 0};
      if (dg * 8 < A.vdim) {
        const bf16_t* src = rows + (u64)(k0 + 2 * kp) * A.ld + voff + dg * 8;
        if (k0 + 2 * kp < cnt) a = *(const u32x4*)src;
        if (k0 + 2 * kp + 1 < cnt) b = *(const u32x4*)(src + A.ld);
      }
      const u32 blk = kp >> 2, off = (kp & 3) * 4;
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        const u32 row = dg * 8 + e, sh = (e & 1) * 16;
        *(u32*)(ldsX + row * 128 + ((blk ^ swz(row)) << 4) + off) =
            ((a[e >> 1] >> sh) & 0xFFFFu) |
            (((b[e >> 1] >> sh) & 0xFFFFu) << 16);
      }
    }
    __syncthreads();
#pragma unroll
    for (int k2 = 0; k2 < 2; ++k2) {
      const u32 blk = k2 * 4 + l4;
      s16x8 b[NTW];
#pragma unroll
      for (int j = 0; j < NTW; ++j) {
        const u32 row = (wave * NTW + j) * 16 + l15;
        b[j] = *(const s16x8*)(ldsX + row * 128 + ((blk ^ swz(row)) << 4));
      }
#pragma unroll
      for (int mt = 0; mt < 4; ++mt) {
        const int po = (mt * 16 + l15) * PROW + (k2 * 32 + l4 * 8) * 2;
        const s16x8 ah = *(const s16x8*)(ldsPh + po);
        const s16x8 al = *(const s16x8*)(ldsPl + po);
#pragma unroll
        for (int j = 0; j < NTW; ++j) {
          acc[mt][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
              ah, b[j], acc[mt][j], 0, 0, 0);
          acc[mt][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
              al, b[j], acc[mt][j], 0, 0, 0);
        }
      }
    }
  }

  // ---- denominator: 8 threads a row for n_c . q -----------------------------
  {
    const int t = tid >> 3, part = tid & 7;
    float d = 0.f;
    if (inter) {
      const float* nc = A.nws + (cid * A.heads + h) * A.DP;
      const unsigned short* q = (const unsigned short*)(ldsQ + t * KROW);
      for (int e = part; e < A.dim; e += 8)
        d = fmaf(bf16_bits_to_f32(q[e]), nc[e], d);
    }
    d += __shfl_xor(d, 1, 64);
    d += __shfl_xor(d, 2, 64);
    d += __shfl_xor(d, 4, 64);
    if (part == 0) {
      const float den = denp[t] + denp[64 + t] + Ct[t] * d;
      sc[t] = 1.f / (fmaxf(fabsf(den), expf(-Mt[t])) + 1e-6f);
    }
  }
  __syncthreads();
  // ---- head norm, weight, gate ----------------------------------------------
#pragma unroll
  for (int mt = 0; mt < 4; ++mt)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int t = mt * 16 + l4 * 4 + r;
      const float f = sc[t];
      float ss = 0.f;
#pragma unroll
      for (int j = 0; j < NTW; ++j) {
        acc[mt][j][r] *= f;
        ss = fmaf(acc[mt][j][r], acc[mt][j][r], ss);
      }
#pragma unroll
      for (int o = 8; o > 0; o >>= 1) ss += __shfl_xor(ss, o, 64);
      if (l15 == 0) red[wave * 64 + t] = ss;
    }
  __syncthreads();
  if (tid < 64) {
    float ss = 0.f;
#pragma unroll
    for (int w = 0; w < 8; ++w) ss += red[w * 64 + tid];
    sc[tid] = 1.f / sqrtf(ss / (float)A.vdim + A.eps);
  }
  __syncthreads();
  const u64 goff = voff + (u64)A.heads * A.vdim;
#pragma unroll
  for (int mt = 0; mt < 4; ++mt)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int t = mt * 16 + l4 * 4 + r;
      if (q0 + t >= cnt) continue;
      const float f = sc[t];
      const bf16_t* g = rows + (u64)(q0 + t) * A.ld + goff;
      bf16_t* o = A.out + ((u64)(n0 + q0 + t) * A.heads + h) * A.vdim;
#pragma unroll
      for (int j = 0; j < NTW; ++j) {
        const int v = (wave * NTW + j) * 16 + l15;
        if (v < A.vdim)
          stf(o + v, acc[mt][j][r] * f * A.norm_w[h * A.vdim + v] *
                         sigmoid_f(ldf(g + v)));
      }
    }
}

template <int KS, int NTW>
hipError_t launch_out(const SeqView& sv, const CArgs& A, int max_count,
                      hipStream_t stream) {
  constexpr size_t lds = out_lds<KS, NTW>();
  static bool set = false;
  if (!set && lds > 64 * 1024) {
    LFMQ_CHECK_HIP(hipFuncSetAttribute(
        (const void*)mlstm_out_kernel<KS, NTW>,
        hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds));
    set = true;
  }
  hipLaunchKernelGGL((mlstm_out_kernel<KS, NTW>),
                     dim3((max_count + 63) / 64, A.heads, sv.b), dim3(512),
                     lds, stream, sv, A);
  return hipGetLastError();
}

}  // namespace

// row layout [q | k | v | gate]; false: the token-by-token kernel's shape
bool lfmq_mlstm_chunk_ok(const void* qkv, long ld, int dim, int vdim) {
  return ((u64)qkv & 15) == 0 && ld % 8 == 0 && dim % 8 == 0 &&
         vdim % 8 == 0 && dim <= 256 && vdim <= 512;
}

// ws: chunks * H * 2 * VP * DP bf16, nws: chunks * H * DP floats with DP, VP
// the sizes rounded up to 64; gws: 3 * H * N floats; L 64, 128 or 256
hipError_t lfmq_mlstm_chunk(const void* qkv, long ld, const void* gates,
                            const SeqView& sv, const void* turn,
                            const void* chunk_base, void* S, void* nm,
                            void* ws, void* nws, void* gws,
                            const void* norm_w, void* out, int heads, int dim,
                            int vdim, float cap, float eps, int L,
                            int max_count, hipStream_t stream) {
  if (L != 64 && L != 128 && L != 256) return hipErrorInvalidValue;
  float* g = (float*)gws;
  const u64 hn = (u64)heads * sv.n;
  CArgs A{(const bf16_t*)qkv, (u64)ld, g, g + hn, g + 2 * hn,
          (const i32*)turn, (const i32*)chunk_base, (float*)S, (float*)nm,
          (unsigned short*)ws, (float*)nws, (const float*)norm_w,
          (bf16_t*)out, heads, dim, vdim, L, (dim + 63) / 64 * 64,
          (vdim + 63) / 64 * 64, eps};
  hipLaunchKernelGGL(mlstm_gate_scan_kernel, dim3(heads, sv.b), dim3(GT), 0,
                     stream, (const float*)gates, sv, (const i32*)turn,
                     (float*)nm, g, g + hn, g + 2 * hn, heads, dim, cap,
                     L / 64);
  LFMQ_CHECK_HIP(hipGetLastError());
  hipLaunchKernelGGL(mlstm_states_kernel,
                     dim3((A.DP / 64) * (A.VP / 64), heads, sv.b), dim3(256),
                     0, stream, sv, A);
  LFMQ_CHECK_HIP(hipGetLastError());
  const int ks = (dim + 31) / 32, ntw = (vdim + 127) / 128;
#define GO(K, N) return launch_out<K, N>(sv, A, max_count, stream)
#define GON(K)                                                               \
  do {                                                                       \
    if (ntw <= 1) GO(K, 1);                                                  \
    if (ntw <= 2) GO(K, 2);                                                  \
    GO(K, 4);                                                                \
  } while (0)
  if (ks <= 2) GON(2);
  if (ks <= 4) GON(4);
  GON(8);
#undef GON
#undef GO
}
