// Mixture of experts on packed rows, weights in the model's dtype.
//
// moe_route: router logits of h in fp32 (one pass also yields the shared
//   expert's gate), sigmoid scores, the `top` largest of each token, and the
//   sort of (token, choice) pairs by expert:
//     src[slot] token, weight[slot] score, pos[token, choice] = slot,
//     tiles[t] = {expert, first slot, slots} of at most `bm` slots, expert
//     -1 past the last one.  Everything stays on the device.
// moe_glu:  act[slot] = glu(weight * (W_gate h), weight * (W_up h)), since
//   the weight scales the expert's input and the products are linear;
//   g = min(g, limit), u = clamp(u), glu = g sigmoid(alpha g) (u + beta)
// moe_down: rows[slot] = W_down act[slot]; the sum over a token's slots is
//   part of the norm that reads them.
//
// Three forms of the two products: 128-row tiles through LDS (prompts),
// 16-row tiles whose waves split the inner dimension and stream the weights
// past registers (few rows an expert: decoding), and any size, 16 or 32 bit.
#include "seq_common.h"

namespace {

// ---------------------------------------------------------------------------
// routing
// ---------------------------------------------------------------------------

constexpr int RT = 1024, RW = RT / 64, RROWS = 16;
constexpr int EG = 32;      // experts a pass over the router's matrix

struct RouteArgs {
  const void *h, *w;      // w [E + has_sg, width]
  i32* ids;               // [n, top]
  float* score;           // [n, top]
  float* sg;              // [n] or null
  i32 *src, *pos;
  float* weight;
  i32* tiles;             // [max_tiles, 3]
  int n, width, E, top, bm, max_tiles;
};

// one workgroup; cnt and offs [E] in LDS
__device__ void sort_pairs(const RouteArgs& A, int* cnt, int* offs) {
  const int tid = threadIdx.x, tpb = blockDim.x, pairs = A.n * A.top;
  for (int e = tid; e < A.E; e += tpb) cnt[e] = 0;
  __syncthreads();
  for (int p = tid; p < pairs; p += tpb) atomicAdd(cnt + A.ids[p], 1);
  __syncthreads();
  if (tid < 64) {
    int base = 0, tbase = 0;
    for (int e0 = 0; e0 < A.E; e0 += 64) {
      const int e = e0 + tid;
      const int c = e < A.E ? cnt[e] : 0, t = (c + A.bm - 1) / A.bm;
      int ci = c, ti = t;
#pragma unroll
      for (int o = 1; o < 64; o <<= 1) {
        const int cu = __shfl_up(ci, o, 64), tu = __shfl_up(ti, o, 64);
        if (tid >= o) {
          ci += cu;
          ti += tu;
        }
      }
      const int first = base + ci - c, tfirst = tbase + ti - t;
      if (e < A.E) {
        offs[e] = first;
        for (int i = 0; i < t && tfirst + i < A.max_tiles; ++i) {
          i32* o = A.tiles + 3 * (tfirst + i);
          o[0] = e;
          o[1] = first + i * A.bm;
          o[2] = min(A.bm, c - i * A.bm);
        }
      }
      base += __shfl(ci, 63, 64);
      tbase += __shfl(ti, 63, 64);
    }
    for (int i = tbase + tid; i < A.max_tiles; i += 64) A.tiles[3 * i] = -1;
  }
  __syncthreads();
  for (int p = tid; p < pairs; p += tpb) {
    const int slot = atomicAdd(offs + A.ids[p], 1);
    A.src[slot] = p / A.top;
    A.weight[slot] = A.score[p];
    A.pos[p] = slot;
  }
}

__global__ __launch_bounds__(1024) void moe_sort_kernel(RouteArgs A) {
  extern __shared__ int shi[];
  sort_pairs(A, shi, shi + A.E);
}

template <typename T, bool MF>
__global__ __launch_bounds__(RT) void moe_route_kernel(RouteArgs A) {
  extern __shared__ float sh[];
  const int E1 = A.E + (A.sg != nullptr);
  float* lg = sh;                      // [RROWS][E1]
  float* red = sh + RROWS * E1;        // MF: [RW][16][EG]
  const int r0 = blockIdx.x * RROWS;
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  const T* h = (const T*)A.h;
  const T* w = (const T*)A.w;
  if constexpr (MF) {
    const int l15 = lane & 15, l4 = lane >> 4;
    const T* hr = h + (u64)min(r0 + l15, A.n - 1) * A.width;
    const s16x8 z8 = {0, 0, 0, 0, 0, 0, 0, 0};
    for (int e0 = 0; e0 < E1; e0 += EG) {
      f32x4 acc[EG / 16] = {};
      const T* wr[EG / 16];
#pragma unroll
      for (int j = 0; j < EG / 16; ++j)
        wr[j] = w + (u64)min(e0 + j * 16 + l15, E1 - 1) * A.width;
      constexpr int U = 4;       // steps loaded ahead of their products
      for (int k = wave * 32; k < A.width; k += U * RW * 32) {
        s16x8 a[U], b[U][EG / 16];
#pragma unroll
        for (int i = 0; i < U; ++i) {
          const int kk = k + i * RW * 32 + l4 * 8;
          const bool ok = kk < A.width;
          a[i] = ok ? *(const s16x8*)(hr + kk) : z8;
#pragma unroll
          for (int j = 0; j < EG / 16; ++j)
            b[i][j] = ok ? *(const s16x8*)(wr[j] + kk) : z8;
        }
#pragma unroll
        for (int i = 0; i < U; ++i)
#pragma unroll
          for (int j = 0; j < EG / 16; ++j)
            acc[j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a[i], b[i][j],
                                                             acc[j], 0, 0, 0);
      }
      __syncthreads();
#pragma unroll
      for (int j = 0; j < EG / 16; ++j)
#pragma unroll
        for (int r = 0; r < 4; ++r)
          red[(wave * 16 + l4 * 4 + r) * EG + j * 16 + l15] = acc[j][r];
      __syncthreads();
      for (int id = tid; id < 16 * EG; id += RT) {
        const int e = e0 + id % EG;
        if (e >= E1) continue;
        float v = 0.f;
#pragma unroll
        for (int g = 0; g < RW; ++g) v += red[g * 16 * EG + id];
        lg[id / EG * E1 + e] = v;
      }
    }
  } else {
    for (int id = wave; id < RROWS * E1; id += RW) {
      const int r = id / E1, e = id % E1;
      if (r0 + r >= A.n) break;
      const T* hr = h + (u64)(r0 + r) * A.width;
      const T* wr = w + (u64)e * A.width;
      float v = 0.f;
      for (int k = lane; k < A.width; k += 64)
        v = fmaf(ldf(hr + k), ldf(wr + k), v);
      v = wave_reduce_sum(v);
      if (lane == 0) lg[id] = v;
    }
  }
  __syncthreads();
  for (int r = wave; r < RROWS; r += RW) {
    const int row = r0 + r;
    if (row >= A.n) break;
    float* z = lg + r * E1;
    if (lane == 0 && A.sg != nullptr) A.sg[row] = sigmoid_f(z[A.E]);
    // a lane watches experts lane, lane + 64, ...; a chosen one drops out
    for (int k = 0; k < A.top; ++k) {
      float best = -INFINITY;
      int id = A.E;
      for (int e = lane; e < A.E; e += 64)
        if (z[e] > best) {
          best = z[e];
          id = e;
        }
#pragma unroll
      for (int o = 32; o > 0; o >>= 1) {
        const float v = __shfl_xor(best, o, 64);
        const int j = __shfl_xor(id, o, 64);
        if (v > best || (v == best && j < id)) {
          best = v;
          id = j;
        }
      }
      id = min(id, A.E - 1);
      if (lane == 0) {
        A.ids[(u64)row * A.top + k] = id;
        A.score[(u64)row * A.top + k] = sigmoid_f(best);
      }
      if (lane == (id & 63)) z[id] = -INFINITY;
    }
  }
  if (gridDim.x == 1) {       // few rows: sort right here
    __syncthreads();
    int* cnt = (int*)sh;
    sort_pairs(A, cnt, cnt + A.E);
  }
}

// ---------------------------------------------------------------------------
// products
// ---------------------------------------------------------------------------

struct GemmArgs {
  const void *a, *w;      // a [*, K]; w [E, GLU ? 2 N : N, K]
  const i32* src;         // row of a for a slot, or null: the slot itself
  const float* weight;    // GLU: per slot, or null
  const i32* tiles;
  void* out;              // [slots, N]
  int N, K;
  float limit, alpha, beta;
};

// T: the storage type (16-bit results take the hardware's exponential)
template <typename T>
__device__ __forceinline__ float glu_f(float g, float u, const GemmArgs& A) {
  g = fminf(g, A.limit);
  u = fminf(fmaxf(u, -A.limit), A.limit);
  const float s = sizeof(T) == 2
                      ? __builtin_amdgcn_rcpf(1.f + __expf(-A.alpha * g))
                      : sigmoid_f(A.alpha * g);
  return g * s * (u + A.beta);
}

// 16 rows x 16 columns; NW waves split K in pairs of 32
template <bool GLU, int NW>
__global__ __launch_bounds__(NW * 64) void moe_rows16(GemmArgs A) {
  constexpr int NB = GLU ? 2 : 1;
  __shared__ float red[NW][NB][16][17];
  const i32* tile = A.tiles + 3 * blockIdx.y;
  const int ex = tile[0];
  if (ex < 0) return;
  const int row0 = tile[1], rows = tile[2];
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  const int l15 = lane & 15, l4 = lane >> 4;
  const int n0 = blockIdx.x * 16, n = min(n0 + l15, A.N - 1);
  const int slot = row0 + min(l15, rows - 1);
  const bf16_t* ar =
      (const bf16_t*)A.a + (u64)(A.src != nullptr ? A.src[slot] : slot) * A.K;
  const bf16_t* w = (const bf16_t*)A.w + (u64)ex * NB * A.N * A.K;
  const bf16_t* wr[NB];
  wr[0] = w + (u64)n * A.K;
  if constexpr (GLU) wr[1] = w + (u64)(A.N + n) * A.K;
  const s16x8 z8 = {0, 0, 0, 0, 0, 0, 0, 0};
  f32x4 acc[NB] = {};
  constexpr int U = 8;           // steps loaded ahead of their products
  for (int k = wave * 64; k < A.K; k += U / 2 * NW * 64) {
    s16x8 a[U], b[U][NB];
#pragma unroll
    for (int i = 0; i < U; ++i) {
      const int kk = k + (i >> 1) * NW * 64 + (i & 1) * 32 + l4 * 8;
      const bool ok = kk < A.K;
      a[i] = ok ? *(const s16x8*)(ar + kk) : z8;
#pragma unroll
      for (int j = 0; j < NB; ++j)
        b[i][j] = ok ? *(const s16x8*)(wr[j] + kk) : z8;
    }
#pragma unroll
    for (int i = 0; i < U; ++i)
#pragma unroll
      for (int j = 0; j < NB; ++j)
        acc[j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a[i], b[i][j], acc[j],
                                                         0, 0, 0);
  }
#pragma unroll
  for (int j = 0; j < NB; ++j)
#pragma unroll
    for (int r = 0; r < 4; ++r) red[wave][j][l4 * 4 + r][l15] = acc[j][r];
  __syncthreads();
  const int i = tid >> 4, c = tid & 15;
  if (tid >= 256 || i >= rows || n0 + c >= A.N) return;
  float v[NB];
#pragma unroll
  for (int j = 0; j < NB; ++j) {
    v[j] = 0.f;
#pragma unroll
    for (int g = 0; g < NW; ++g) v[j] += red[g][j][i][c];
  }
  float o = v[0];
  if constexpr (GLU) {
    const float s = A.weight != nullptr ? A.weight[row0 + i] : 1.f;
    o = glu_f<bf16_t>(s * v[0], s * v[1], A);
  }
  stf((bf16_t*)A.out + (u64)(row0 + i) * A.N + n0 + c, o);
}

// 128 rows x 128 weight rows (GLU: 64 gate and 64 up), 4 waves of 64 x 64,
// K in steps of 64 through two LDS buffers; 16-byte blocks of a 128-byte LDS
// row are XOR-swizzled by the row so that fragment reads spread over banks
constexpr int BM = 128, BN = 128, BK = 64;

template <bool GLU>
__global__ __launch_bounds__(256, 2) void moe_rows128(GemmArgs A) {
  extern __shared__ __attribute__((aligned(16))) char smem[];
  const i32* tile = A.tiles + 3 * blockIdx.y;
  const int ex = tile[0];
  if (ex < 0) return;
  const int row0 = tile[1], rows = tile[2];
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  const int l15 = lane & 15, l4 = lane >> 4;
  const int wm = wave >> 1, wn = wave & 1;
  const int n0 = blockIdx.x * (GLU ? 64 : 128);
  const int wrows = GLU ? 2 * A.N : A.N;
  const bf16_t* w = (const bf16_t*)A.w + (u64)ex * wrows * A.K;
  // staging role: 16-byte column sc of rows sr + 32 i
  const int sr = tid >> 3, sc = tid & 7;
  const bf16_t *ap[4], *bp[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int r = sr + 32 * i;
    const int slot = row0 + min(r, rows - 1);
    ap[i] = (const bf16_t*)A.a +
            (u64)(A.src != nullptr ? A.src[slot] : slot) * A.K;
    int n;
    if constexpr (GLU)
      n = (r < 64 ? 0 : A.N) + min(n0 + (r & 63), A.N - 1);
    else
      n = min(n0 + r, A.N - 1);
    bp[i] = w + (u64)n * A.K;
  }
  u32x4 xa[4], xb[4];
  auto fetch = [&](int k0) {
    const int k = k0 + sc * 8;
    const u32x4 z = {0, 0, 0, 0};
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      xa[i] = k < A.K ? *(const u32x4*)(ap[i] + k) : z;
      xb[i] = k < A.K ? *(const u32x4*)(bp[i] + k) : z;
    }
  };
  auto stage = [&](char* buf) {
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int r = sr + 32 * i, o = r * 128 + ((sc ^ (r & 7)) << 4);
      *(u32x4*)(buf + o) = xa[i];
      *(u32x4*)(buf + BM * 128 + o) = xb[i];
    }
  };
  f32x4 acc[4][4] = {};
  fetch(0);
  stage(smem);
  __syncthreads();
  int cur = 0;
  for (int k0 = 0; k0 < A.K; k0 += BK) {
    const bool more = k0 + BK < A.K;
    if (more) fetch(k0 + BK);
    const char* la = smem + cur * (BM + BN) * 128;
    const char* lb = la + BM * 128;
#pragma unroll
    for (int ks = 0; ks < 2; ++ks) {
      s16x8 af[4], bf[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int r = wm * 64 + i * 16 + l15;
        af[i] = *(const s16x8*)(la + r * 128 + (((ks * 4 + l4) ^ (r & 7)) << 4));
        const int c = GLU ? (i >> 1) * 64 + wn * 32 + (i & 1) * 16 + l15
                          : wn * 64 + i * 16 + l15;
        bf[i] = *(const s16x8*)(lb + c * 128 + (((ks * 4 + l4) ^ (c & 7)) << 4));
      }
#pragma unroll
      for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j)
          acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
              af[i], bf[j], acc[i][j], 0, 0, 0);
    }
    cur ^= 1;
    if (more) stage(smem + cur * (BM + BN) * 128);
    __syncthreads();
  }
#pragma unroll
  for (int i = 0; i < 4; ++i)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int row = wm * 64 + i * 16 + l4 * 4 + r;
      if (row >= rows) continue;
      bf16_t* o = (bf16_t*)A.out + (u64)(row0 + row) * A.N;
      if constexpr (GLU) {
        const float s = A.weight != nullptr ? A.weight[row0 + row] : 1.f;
#pragma unroll
        for (int j = 0; j < 2; ++j) {
          const int n = n0 + wn * 32 + j * 16 + l15;
          if (n < A.N) stf(o + n, glu_f<bf16_t>(s * acc[i][j][r],
                                               s * acc[i][j + 2][r], A));
        }
      } else {
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          const int n = n0 + wn * 64 + j * 16 + l15;
          if (n < A.N) stf(o + n, acc[i][j][r]);
        }
      }
    }
}

// any size: tiles of one row; a wave a column at a time
template <typename T, bool GLU>
__global__ __launch_bounds__(256) void moe_any(GemmArgs A) {
  const i32* tile = A.tiles + 3 * blockIdx.y;
  const int ex = tile[0];
  if (ex < 0) return;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const T* w = (const T*)A.w + (u64)ex * (GLU ? 2 : 1) * A.N * A.K;
  for (int i = 0; i < tile[2]; ++i) {
    const int slot = tile[1] + i;
    const T* a =
        (const T*)A.a + (u64)(A.src != nullptr ? A.src[slot] : slot) * A.K;
    for (int n = blockIdx.x * 64 + wave; n < min(A.N, (int)blockIdx.x * 64 + 64);
         n += 4) {
      float v = 0.f, u = 0.f;
      for (int k = lane; k < A.K; k += 64) {
        const float x = ldf(a + k);
        v = fmaf(x, ldf(w + (u64)n * A.K + k), v);
        if (GLU) u = fmaf(x, ldf(w + (u64)(A.N + n) * A.K + k), u);
      }
      v = wave_reduce_sum(v);
      if (GLU) {
        u = wave_reduce_sum(u);
        const float s = A.weight != nullptr ? A.weight[slot] : 1.f;
        v = glu_f<T>(s * v, s * u, A);
      }
      if (lane == 0) stf((T*)A.out + (u64)slot * A.N + n, v);
    }
  }
}

// the same activation on a fused [gate | up] row
template <typename T, int VEC>
__global__ __launch_bounds__(256) void clamped_glu_kernel(
    const T* __restrict__ gu, T* __restrict__ y, u64 rows, int ff,
    GemmArgs A) {
  const u64 total = rows * ff / VEC;
  const int per = ff / VEC;
  for (u64 id = (u64)blockIdx.x * 256 + threadIdx.x; id < total;
       id += (u64)gridDim.x * 256) {
    const u64 row = id / per;
    const int j = id % per * VEC;
    const T* p = gu + row * 2 * ff + j;
    float g[VEC], u[VEC];
    ldv<T, VEC>(p, g);
    ldv<T, VEC>(p + ff, u);
#pragma unroll
    for (int e = 0; e < VEC; ++e) g[e] = glu_f<T>(g[e], u[e], A);
    stv<T, VEC>(y + row * ff + j, g);
  }
}

template <bool GLU>
hipError_t gemm(const GemmArgs& A, int max_tiles, int bm, bool f32,
                hipStream_t stream) {
  if (max_tiles < 1 || max_tiles > 65535) return hipErrorInvalidValue;
  if (bm == 128 && !f32) {
    const size_t lds = 2 * (BM + BN) * 128;
    const int per = GLU ? 64 : 128;
    hipLaunchKernelGGL(moe_rows128<GLU>,
                       dim3((A.N + per - 1) / per, max_tiles), dim3(256), lds,
                       stream, A);
  } else if (bm == 16 && !f32) {
    const dim3 grid((A.N + 15) / 16, max_tiles);
    if (A.K >= 1024)
      hipLaunchKernelGGL((moe_rows16<GLU, 8>), grid, dim3(512), 0, stream, A);
    else
      hipLaunchKernelGGL((moe_rows16<GLU, 4>), grid, dim3(256), 0, stream, A);
  } else {
    const dim3 grid((A.N + 63) / 64, max_tiles);
    if (f32)
      hipLaunchKernelGGL((moe_any<float, GLU>), grid, dim3(256), 0, stream, A);
    else
      hipLaunchKernelGGL((moe_any<bf16_t, GLU>), grid, dim3(256), 0, stream, A);
  }
  return hipGetLastError();
}

}  // namespace

// tiles [max_tiles, 3]; mfma: width % 8 == 0 and 16-byte rows
hipError_t lfmq_moe_route_sort(const void* h, const void* w, void* ids,
                               void* score, void* sg, void* src, void* weight,
                               void* pos, void* tiles, int n, int width,
                               int E, int top, int bm, int max_tiles,
                               bool mfma, bool f32, hipStream_t stream) {
  RouteArgs A{h, w, (i32*)ids, (float*)score, (float*)sg, (i32*)src,
              (i32*)pos, (float*)weight, (i32*)tiles, n, width, E, top, bm,
              max_tiles};
  const int E1 = E + (sg != nullptr);
  const size_t lds = sizeof(float) * (size_t)(RROWS * E1 + (mfma ? RW * 16 * EG : 0));
  if (lds > 64 * 1024 || top > E) return hipErrorInvalidValue;
  const dim3 grid((n + RROWS - 1) / RROWS), block(RT);
  if (f32)
    hipLaunchKernelGGL((moe_route_kernel<float, false>), grid, block, lds, stream, A);
  else if (mfma)
    hipLaunchKernelGGL((moe_route_kernel<bf16_t, true>), grid, block, lds, stream, A);
  else
    hipLaunchKernelGGL((moe_route_kernel<bf16_t, false>), grid, block, lds, stream, A);
  if (grid.x > 1)
    hipLaunchKernelGGL(moe_sort_kernel, dim3(1), dim3(1024),
                       2 * E * sizeof(int), stream, A);
  return hipGetLastError();
}

hipError_t lfmq_moe_glu(const void* a, const void* w, const void* src,
                        const void* weight, const void* tiles, void* out,
                        int N, int K, float limit, float alpha, float beta,
                        int max_tiles, int bm, bool f32, hipStream_t stream) {
  GemmArgs A{a, w, (const i32*)src, (const float*)weight, (const i32*)tiles,
             out, N, K, limit, alpha, beta};
  return gemm<true>(A, max_tiles, bm, f32, stream);
}

hipError_t lfmq_moe_down(const void* a, const void* w, const void* tiles,
                         void* out, int N, int K, int max_tiles, int bm,
                         bool f32, hipStream_t stream) {
  GemmArgs A{a, w, nullptr, nullptr, (const i32*)tiles, out, N, K, 0.f, 0.f,
             0.f};
  return gemm<false>(A, max_tiles, bm, f32, stream);
}

hipError_t lfmq_clamped_glu(const void* gu, void* y, long rows, int ff,
                            float limit, float alpha, float beta, bool f32,
                            hipStream_t stream) {
  GemmArgs A{};
  A.limit = limit;
  A.alpha = alpha;
  A.beta = beta;
  const bool v4 = ff % 4 == 0 && (((u64)gu | (u64)y) & 15) == 0;
  const u64 want = ((u64)rows * ff / (v4 ? 4 : 1) + 255) / 256;
  const dim3 grid((u32)(want < 8192 ? want : 8192));
#define GO(T, V)                                                             \
  hipLaunchKernelGGL((clamped_glu_kernel<T, V>), grid, dim3(256), 0, stream, \
                     (const T*)gu, (T*)y, (u64)rows, ff, A)
  if (f32) { if (v4) GO(float, 4); else GO(float, 1); }
  else { if (v4) GO(bf16_t, 4); else GO(bf16_t, 1); }
#undef GO
  return hipGetLastError();
}
