// lfmq_seq — torch bindings of the sequence-mixing layers' kernels (packed
// variable-length batches, recurrent states, latent and grouped attention,
// experts) and of the small ops every model shares.  Every entry checks dtypes,
// devices and the sizes that its kernel and grid assume; no fallbacks.
#include <torch/extension.h>
#include <ATen/cuda/CUDAContext.h>
#include <hip/hip_runtime.h>

#include "seq_common.h"

using T_ = torch::Tensor;
using OptT = c10::optional<torch::Tensor>;

hipError_t lfmq_bigram_embed(const void*, const SeqView&, const void*,
                             const void*, const void*, void*, int, long, long,
                             long, long, bool, hipStream_t);
hipError_t lfmq_seq_advance(const void*, const void*, const void*, void*,
                            void*, void*, int, hipStream_t);
hipError_t lfmq_add_norm(void*, const void*, const void*, float, void*, int,
                         int, float, const void*, const void*, void*, int,
                         bool, hipStream_t);
hipError_t lfmq_head_norm_gate(const void*, const void*, long, const void*,
                               void*, long, int, int, float, bool,
                               hipStream_t);
hipError_t lfmq_mlstm_scan(const void*, long, const void*, const SeqView&,
                           const void*, void*, void*, void*, int, int, int,
                           float, bool, hipStream_t);
bool lfmq_mlstm_chunk_ok(const void*, long, int, int);
hipError_t lfmq_mlstm_chunk(const void*, long, const void*, const SeqView&,
                            const void*, const void*, void*, void*, void*,
                            void*, void*, const void*, void*, int, int, int,
                            float, float, int, int, hipStream_t);
hipError_t lfmq_latent_prep(const void*, long, const SeqView&, const void*,
                            const void*, const void*, void*, void*,
                            const void*, int, int, int, int, int, float, bool,
                            hipStream_t);
hipError_t lfmq_latent_ring(const SeqView&, const void*, const void*, void*,
                            void*, int, int, bool, bool, hipStream_t);
hipError_t lfmq_latent_absorb(const void*, const void*, const SeqView&,
                              const void*, void*, int, int, int, int, int,
                              bool, hipStream_t);
hipError_t lfmq_latent_expand(const void*, int, const void*, const void*,
                              const void*, long, void*, int, int, int, int,
                              bool, hipStream_t);
hipError_t lfmq_attn_window_prompt(const void*, const void*, long, long,
                                   const void*, long, const void*, long, long,
                                   const SeqView&, const void*, const void*,
                                   const void*, const void*, long, void*, int,
                                   int, int, int, int, int, float, bool,
                                   hipStream_t);
hipError_t lfmq_attn_window_decode(const void*, const void*, const SeqView&,
                                   void*, int, int, int, int, int, int, float,
                                   bool, hipStream_t);
bool lfmq_attn_latent_decode_mfma_ok(const void*, const void*, int, int);
hipError_t lfmq_attn_latent_decode_mfma(const void*, const void*,
                                        const SeqView&, void*, int, int, int,
                                        int, int, int, float, hipStream_t);
bool lfmq_attn_window_prompt_mfma_ok(const void*, const void*, long,
                                     const void*, long, const void*, long, int,
                                     int, int);
hipError_t lfmq_attn_window_prompt_mfma(
    const void*, const void*, long, const void*, long, const void*, long,
    const SeqView&, const void*, const void*, const void*, const void*, long,
    void*, int, int, int, int, int, int, float, int, hipStream_t);
hipError_t lfmq_post_norm(void*, const void*, const void*, const void*, void*,
                          int, int, float, float, bool, hipStream_t);
hipError_t lfmq_embed_norm(void*, const void*, const void*, const void*,
                           void*, int, int, int, float, bool, hipStream_t);
hipError_t lfmq_post_norm_experts(void*, const void*, const void*, int,
                                  const void*, const void*, const void*,
                                  const void*, void*, int, int, float, float,
                                  bool, hipStream_t);
hipError_t lfmq_qk_prep(const void*, long, const SeqView&, const void*,
                        const void*, const void*, void*, void*, void*, int,
                        int, int, int, int, int, float, bool, hipStream_t);
hipError_t lfmq_attn_grouped(const void*, const void*, const void*,
                             const SeqView&, const void*, void*, long, int,
                             int, int, int, int, float, float, bool,
                             hipStream_t);
bool lfmq_attn_grouped_mfma_ok(const void*, const void*, const void*, int,
                               int);
hipError_t lfmq_attn_grouped_mfma(const void*, const void*, const void*,
                                  const SeqView&, const void*, void*, long,
                                  int, int, int, int, int, float, float, int,
                                  hipStream_t);
int lfmq_attn_grouped_splits(int, int, int, int);
hipError_t lfmq_attn_grouped_decode(const void*, const void*, const void*,
                                    const SeqView&, const void*, void*, void*,
                                    long, int, int, int, int, int, int, float,
                                    float, hipStream_t);
bool lfmq_lru_mfma_ok(const void*, int, int);
hipError_t lfmq_gated_lru(const SeqView&, const void*, const void*, long,
                          const void*, const void*, const void*, const void*,
                          const void*, const void*, const void*, void*, void*,
                          void*, long, int, int, int, float, float, void*,
                          void*, void*, const void*, int, bool, bool, bool,
                          hipStream_t);
hipError_t lfmq_moe_route_sort(const void*, const void*, void*, void*, void*,
                               void*, void*, void*, void*, int, int, int, int,
                               int, int, bool, bool, hipStream_t);
hipError_t lfmq_moe_glu(const void*, const void*, const void*, const void*,
                        const void*, void*, int, int, float, float, float,
                        int, int, bool, hipStream_t);
hipError_t lfmq_moe_down(const void*, const void*, const void*, void*, int,
                         int, int, int, bool, hipStream_t);
hipError_t lfmq_clamped_glu(const void*, void*, long, int, float, float,
                            float, bool, hipStream_t);
hipError_t lfmq_silu_mul_fused(const void*, void*, long, int, hipStream_t);
hipError_t lfmq_silu_mul_any(const void*, void*, long, int, bool,
                             hipStream_t);
hipError_t lfmq_argmax_rows(const void*, void*, void*, void*, int, int,
                            hipStream_t);
hipError_t lfmq_argmax_rows_any(const void*, void*, void*, void*, int, int,
                                bool, hipStream_t);
hipError_t lfmq_advance_record(void*, void*, const void*, void*, int, int,
                               hipStream_t);

namespace {

#define CHECK_HIP(call)                                                     \
  do {                                                                      \
    hipError_t e = (call);                                                  \
    TORCH_CHECK(e == hipSuccess, "lfmq HIP error: ", hipGetErrorString(e)); \
  } while (0)

hipStream_t stream() {
  return (hipStream_t)at::cuda::getCurrentCUDAStream().stream();
}

void check(const T_& t, torch::ScalarType dt, const char* name) {
  TORCH_CHECK(t.is_cuda() && t.is_contiguous(), name,
              " must be a contiguous GPU tensor");
  TORCH_CHECK(t.scalar_type() == dt, name, " has dtype ", t.scalar_type(),
              ", expected ", dt);
}

bool storage(const T_& t, const char* name) {
  TORCH_CHECK(t.is_cuda(), name, " must be on GPU");
  const bool f32 = t.scalar_type() == torch::kFloat32;
  TORCH_CHECK(f32 || t.scalar_type() == torch::kBFloat16, name,
              " must be bf16 or fp32");
  return f32;
}

// rows of a projection output: unit column stride, any row stride
long row_stride(const T_& t, long cols, const char* name) {
  TORCH_CHECK(t.dim() == 2 && t.stride(1) == 1 && t.size(1) >= cols, name,
              " must be row-major with at least ", cols, " columns");
  return t.stride(0);
}

SeqView view(const T_& seq, const T_& cu, const T_& slots, const T_& lens) {
  check(seq, torch::kInt32, "seq");
  check(cu, torch::kInt32, "cu");
  check(slots, torch::kInt32, "slots");
  check(lens, torch::kInt32, "lens");
  TORCH_CHECK(cu.numel() == slots.numel() + 1, "cu must have b + 1 entries");
  TORCH_CHECK(seq.numel() > 0 && slots.numel() > 0, "empty step");
  TORCH_CHECK(slots.numel() <= 65535, "too many sequences in a step");
  return SeqView{(const i32*)seq.data_ptr(), (const i32*)cu.data_ptr(),
                 (const i32*)slots.data_ptr(), (const i32*)lens.data_ptr(),
                 (int)slots.numel(), (int)seq.numel()};
}

T_ bigram_embed(T_ tok, T_ seq, T_ cu, T_ slots, T_ lens, T_ prev, T_ embed,
                T_ bigram, long mul_prev, long mul_cur) {
  const SeqView sv = view(seq, cu, slots, lens);
  check(tok, torch::kInt64, "tok");
  check(prev, torch::kInt32, "prev");
  const bool f32 = storage(embed, "embed");
  check(embed, embed.scalar_type(), "embed");
  check(bigram, embed.scalar_type(), "bigram");
  TORCH_CHECK(tok.numel() == sv.n && bigram.size(1) == embed.size(1) &&
                  prev.numel() == lens.numel() && bigram.size(0) >= 2 &&
                  mul_prev >= 0 && mul_cur >= 0,
              "bigram_embed: shape mismatch");
  auto x = torch::empty({sv.n, embed.size(1)},
                        embed.options().dtype(torch::kFloat32));
  CHECK_HIP(lfmq_bigram_embed(tok.data_ptr(), sv, prev.data_ptr(),
                              embed.data_ptr(), bigram.data_ptr(),
                              x.data_ptr(), (int)embed.size(1), embed.size(0),
                              bigram.size(0) - 1, mul_prev, mul_cur, f32,
                              stream()));
  return x;
}

void seq_advance(T_ tok, T_ cu, T_ slots, T_ lens, T_ prev, T_ turn) {
  check(tok, torch::kInt64, "tok");
  check(cu, torch::kInt32, "cu");
  check(slots, torch::kInt32, "slots");
  for (auto& t : {lens, prev, turn}) check(t, torch::kInt32, "slot state");
  TORCH_CHECK(cu.numel() == slots.numel() + 1 &&
                  lens.numel() == prev.numel() &&
                  lens.numel() == turn.numel(),
              "seq_advance: shape mismatch");
  CHECK_HIP(lfmq_seq_advance(tok.data_ptr(), cu.data_ptr(), slots.data_ptr(),
                             lens.data_ptr(), prev.data_ptr(),
                             turn.data_ptr(), (int)slots.numel(), stream()));
}

// returns {h, side projection or an empty tensor}
std::vector<T_> add_norm(T_ x, OptT y, T_ w, double bias, double eps, OptT wp,
                         OptT bp, bool out_f32) {
  check(x, torch::kFloat32, "x");
  check(w, torch::kFloat32, "norm weight");
  const long n = x.size(0), width = x.size(1);
  TORCH_CHECK(x.dim() == 2 && w.numel() == width, "add_norm: shape mismatch");
  const auto dt = out_f32 ? torch::kFloat32 : torch::kBFloat16;
  const void* yp = nullptr;
  if (y.has_value()) {
    check(*y, dt, "y");
    TORCH_CHECK(y->numel() == n * width, "add_norm: y shape mismatch");
    yp = y->data_ptr();
  }
  auto h = torch::empty({n, width}, x.options().dtype(dt));
  T_ p = torch::empty({0}, x.options());
  const void *wpp = nullptr, *bpp = nullptr;
  long np = 0;
  if (wp.has_value()) {
    check(*wp, dt, "side weight");
    TORCH_CHECK(bp.has_value(), "side projection needs a bias");
    check(*bp, torch::kFloat32, "side bias");
    np = wp->size(0);
    TORCH_CHECK(wp->size(1) == width && bp->numel() == np,
                "side projection shape mismatch");
    p = torch::empty({n, np}, x.options());
    wpp = wp->data_ptr();
    bpp = bp->data_ptr();
  }
  CHECK_HIP(lfmq_add_norm(x.data_ptr(), yp, w.data_ptr(), (float)bias,
                          h.data_ptr(), (int)n, (int)width, (float)eps, wpp,
                          bpp, p.data_ptr(), (int)np, out_f32, stream()));
  return {h, p};
}

T_ head_norm_gate(T_ o, T_ g, T_ w, double eps) {
  check(o, torch::kFloat32, "o");
  check(w, torch::kFloat32, "weight");
  TORCH_CHECK(o.dim() == 3, "o must be [rows, heads, v]");
  const long n = o.size(0), H = o.size(1), V = o.size(2);
  const bool f32 = storage(g, "gate");
  const long ld = row_stride(g, H * V, "gate");
  TORCH_CHECK(g.size(0) == n && w.numel() == H * V, "gate shape mismatch");
  auto out = torch::empty({n, H * V}, g.options());
  CHECK_HIP(lfmq_head_norm_gate(o.data_ptr(), g.data_ptr(), ld, w.data_ptr(),
                                out.data_ptr(), n, (int)H, (int)V, (float)eps,
                                f32, stream()));
  return out;
}

void check_mlstm(const T_& qkv, const T_& gates, const SeqView& sv,
                 const T_& lens, const T_& turn, const T_& S, const T_& nm) {
  check(gates, torch::kFloat32, "gates");
  check(turn, torch::kInt32, "turn");
  check(S, torch::kFloat32, "S");
  check(nm, torch::kFloat32, "nm");
  TORCH_CHECK(S.dim() == 4, "S must be [slots, heads, dim, vdim]");
  const long slots = S.size(0), H = S.size(1), dim = S.size(2);
  TORCH_CHECK(nm.numel() == slots * 2 * H * (dim + 1) &&
                  turn.numel() == slots && lens.numel() == slots &&
                  gates.numel() == sv.n * 2 * H && qkv.size(0) == sv.n,
              "mlstm: shape mismatch");
}

// qkv rows: [q (H dim) | k (H dim) | v (H vdim) | ...]; gates [N, 2H] raw
T_ mlstm_scan(T_ qkv, T_ gates, T_ seq, T_ cu, T_ slots, T_ lens, T_ turn,
              T_ S, T_ nm, double cap) {
  const SeqView sv = view(seq, cu, slots, lens);
  check_mlstm(qkv, gates, sv, lens, turn, S, nm);
  const long H = S.size(1), dim = S.size(2), V = S.size(3);
  const bool f32 = storage(qkv, "qkv");
  const long ld = row_stride(qkv, H * (2 * dim + V), "qkv");
  auto out = torch::empty({sv.n, H, V}, S.options());
  CHECK_HIP(lfmq_mlstm_scan(qkv.data_ptr(), ld, gates.data_ptr(), sv,
                            turn.data_ptr(), S.data_ptr(), nm.data_ptr(),
                            out.data_ptr(), (int)H, (int)dim, (int)V,
                            (float)cap, f32, stream()));
  return out;
}

// whether the chunk kernels take this projection's shape
bool mlstm_chunk_ok(T_ qkv, T_ S) {
  return qkv.scalar_type() == torch::kBFloat16 && qkv.dim() == 2 &&
         qkv.stride(1) == 1 &&
         lfmq_mlstm_chunk_ok(qkv.data_ptr(), qkv.stride(0), (int)S.size(2),
                             (int)S.size(3));
}

// qkv rows [q | k | v | gate]; chunk_base [b] first chunk of each sequence,
// `chunks` in all, L tokens each.  Returns the normed and gated [N, H vdim].
T_ mlstm_chunk(T_ qkv, T_ gates, T_ seq, T_ cu, T_ slots, T_ lens, T_ turn,
               T_ S, T_ nm, double cap, T_ norm_w, double eps, T_ chunk_base,
               long chunks, long L, long max_count) {
  const SeqView sv = view(seq, cu, slots, lens);
  check_mlstm(qkv, gates, sv, lens, turn, S, nm);
  check(norm_w, torch::kFloat32, "norm weight");
  check(chunk_base, torch::kInt32, "chunk_base");
  const long H = S.size(1), dim = S.size(2), V = S.size(3);
  TORCH_CHECK(mlstm_chunk_ok(qkv, S), "mlstm_chunk: shape not supported");
  const long ld = row_stride(qkv, 2 * H * (dim + V), "qkv");
  TORCH_CHECK(norm_w.numel() == H * V && chunk_base.numel() == sv.b &&
                  chunks >= sv.b && max_count >= 1,
              "mlstm_chunk: shape mismatch");
  const long DP = (dim + 63) / 64 * 64, VP = (V + 63) / 64 * 64;
  auto f = S.options();
  auto ws = torch::empty({chunks * H * 2 * VP * DP}, qkv.options());
  auto nws = torch::empty({chunks * H * DP}, f);
  auto gws = torch::empty({3 * H * sv.n}, f);
  auto out = torch::empty({sv.n, H * V}, qkv.options());
  CHECK_HIP(lfmq_mlstm_chunk(
      qkv.data_ptr(), ld, gates.data_ptr(), sv, turn.data_ptr(),
      chunk_base.data_ptr(), S.data_ptr(), nm.data_ptr(), ws.data_ptr(),
      nws.data_ptr(), gws.data_ptr(), norm_w.data_ptr(), out.data_ptr(),
      (int)H, (int)dim, (int)V, (float)cap, (float)eps, (int)L,
      (int)max_count, stream()));
  return out;
}

// dst_row given: rows of `dst` [rows, rank + rot]; else dst is the ring
// [slots, cap, rank + rot].  Returns the normed query latent.
T_ latent_prep(T_ in, T_ seq, T_ cu, T_ slots, T_ lens, T_ wq, T_ wkv,
               T_ inv_freq, T_ dst, OptT dst_row, double eps) {
  const SeqView sv = view(seq, cu, slots, lens);
  check(wq, torch::kFloat32, "query latent norm");
  check(wkv, torch::kFloat32, "kv latent norm");
  check(inv_freq, torch::kFloat32, "inv_freq");
  const bool f32 = storage(in, "in");
  check(dst, in.scalar_type(), "dst");
  const long q_rank = wq.numel(), rank = wkv.numel();
  const long rot = dst.size(-1) - rank, rot_dims = 2 * inv_freq.numel();
  const long ld = row_stride(in, q_rank + rank + rot, "in");
  TORCH_CHECK(rot >= rot_dims && in.size(0) == sv.n,
              "latent_prep: shape mismatch");
  const void* dr = nullptr;
  long cap = 1;
  if (dst_row.has_value()) {
    check(*dst_row, torch::kInt32, "dst_row");
    TORCH_CHECK(dst_row->numel() == sv.b && dst.dim() == 2 &&
                    dst.size(0) >= sv.n,
                "latent_prep: key buffer mismatch");
    dr = dst_row->data_ptr();
  } else {
    TORCH_CHECK(dst.dim() == 3 && dst.size(0) == lens.numel(),
                "latent_prep: ring mismatch");
    cap = dst.size(1);
  }
  auto cq = torch::empty({sv.n, q_rank}, in.options());
  CHECK_HIP(lfmq_latent_prep(in.data_ptr(), ld, sv, wq.data_ptr(),
                             wkv.data_ptr(), inv_freq.data_ptr(),
                             cq.data_ptr(), dst.data_ptr(), dr, (int)cap,
                             (int)q_rank, (int)rank, (int)rot, (int)rot_dims,
                             (float)eps, f32, stream()));
  return cq;
}

void latent_ring(T_ seq, T_ cu, T_ slots, T_ lens, T_ own_row, T_ prior,
                 T_ buf, T_ ring, bool load) {
  const SeqView sv = view(seq, cu, slots, lens);
  check(own_row, torch::kInt32, "own_row");
  check(prior, torch::kInt32, "prior");
  const bool f32 = storage(ring, "ring");
  check(ring, ring.scalar_type(), "ring");
  check(buf, ring.scalar_type(), "buf");
  TORCH_CHECK(ring.dim() == 3 && buf.dim() == 2 &&
                  buf.size(1) == ring.size(2) && own_row.numel() == sv.b &&
                  prior.numel() == sv.b && ring.size(0) == lens.numel(),
              "latent_ring: shape mismatch");
  CHECK_HIP(lfmq_latent_ring(sv, own_row.data_ptr(), prior.data_ptr(),
                             buf.data_ptr(), ring.data_ptr(),
                             (int)ring.size(1), (int)ring.size(2), load, f32,
                             stream()));
}

// q [b, H * (dim + rot)], w [H, dim, rank] -> [b, H, rank + rot]
T_ latent_absorb(T_ q, T_ w, T_ seq, T_ cu, T_ slots, T_ lens, T_ inv_freq,
                 long rot) {
  const SeqView sv = view(seq, cu, slots, lens);
  const bool f32 = storage(q, "q");
  check(q, q.scalar_type(), "q");
  check(w, q.scalar_type(), "w");
  check(inv_freq, torch::kFloat32, "inv_freq");
  const long H = w.size(0), dim = w.size(1), rank = w.size(2);
  TORCH_CHECK(sv.n == sv.b, "one token per sequence expected");
  TORCH_CHECK(q.numel() == sv.b * H * (dim + rot) &&
                  2 * inv_freq.numel() <= rot,
              "latent_absorb: shape mismatch");
  auto out = torch::empty({sv.b, H, rank + rot}, q.options());
  CHECK_HIP(lfmq_latent_absorb(q.data_ptr(), w.data_ptr(), sv,
                               inv_freq.data_ptr(), out.data_ptr(), (int)H,
                               (int)dim, (int)rot,
                               (int)(2 * inv_freq.numel()), (int)rank, f32,
                               stream()));
  return out;
}

// part [b, splits, H, rank + 2], w [H, rank, vdim] -> gated [b, H * vdim]
T_ latent_expand(T_ part, T_ sink, T_ w, T_ g) {
  check(part, torch::kFloat32, "part");
  check(sink, torch::kFloat32, "sink");
  const bool f32 = storage(w, "w");
  check(w, w.scalar_type(), "w");
  const long b = part.size(0), splits = part.size(1), H = w.size(0);
  const long rank = w.size(1), vdim = w.size(2);
  const long ld = row_stride(g, H * vdim, "gate");
  TORCH_CHECK(part.dim() == 4 && part.size(2) == H &&
                  part.size(3) == rank + 2 && sink.numel() == H &&
                  g.size(0) == b && g.scalar_type() == w.scalar_type(),
              "latent_expand: shape mismatch");
  auto out = torch::empty({b, H * vdim}, w.options());
  CHECK_HIP(lfmq_latent_expand(part.data_ptr(), (int)splits, sink.data_ptr(),
                               w.data_ptr(), g.data_ptr(), ld, out.data_ptr(),
                               (int)b, (int)H, (int)rank, (int)vdim, f32,
                               stream()));
  return out;
}

// q [N, H * (d1 + d2)]; kv [rows, H * d1 + H * dv] up-projected keys and
// values; lat [rows, rank + d2] whose tail is the shared key part
T_ attn_window_prompt(T_ q, T_ kv, T_ lat, T_ seq, T_ cu, T_ slots, T_ lens,
                      T_ own_row, T_ inv_freq, T_ sink, T_ g, long d1, long d2,
                      long dv, long window, double scale, long max_count,
                      bool general) {
  const SeqView sv = view(seq, cu, slots, lens);
  const bool f32 = storage(q, "q");
  const auto dt = q.scalar_type();
  check(q, dt, "q");
  check(kv, dt, "kv");
  check(lat, dt, "lat");
  check(own_row, torch::kInt32, "own_row");
  check(inv_freq, torch::kFloat32, "inv_freq");
  check(sink, torch::kFloat32, "sink");
  const long H = sink.numel();
  const long ldg = row_stride(g, H * dv, "gate");
  TORCH_CHECK(q.numel() == sv.n * H * (d1 + d2) && window > 0 &&
                  kv.size(1) == H * (d1 + dv) && kv.size(0) == lat.size(0) &&
                  kv.size(0) >= sv.n && lat.size(1) >= d2 &&
                  g.size(0) == sv.n && g.scalar_type() == dt &&
                  own_row.numel() == sv.b && 2 * inv_freq.numel() <= d2,
              "attn_window_prompt: shape mismatch");
  auto out = torch::empty({sv.n, H * dv}, q.options());
  const long ld = kv.size(1), ll = lat.size(1);
  const size_t es = q.element_size();
  const void* k2 = (const char*)lat.data_ptr() + (ll - d2) * es;
  const void* vp = (const char*)kv.data_ptr() + H * d1 * es;
  if (!f32 && !general &&
      lfmq_attn_window_prompt_mfma_ok(q.data_ptr(), kv.data_ptr(), ld, k2, ll,
                                      vp, ld, (int)d1, (int)d2, (int)dv)) {
    CHECK_HIP(lfmq_attn_window_prompt_mfma(
        q.data_ptr(), kv.data_ptr(), ld, k2, ll, vp, ld, sv,
        own_row.data_ptr(), inv_freq.data_ptr(), sink.data_ptr(),
        g.data_ptr(), ldg, out.data_ptr(), (int)H, (int)d1, (int)d2,
        (int)(2 * inv_freq.numel()), (int)dv, (int)window, (float)scale,
        (int)max_count, stream()));
    return out;
  }
  CHECK_HIP(lfmq_attn_window_prompt(
      q.data_ptr(), kv.data_ptr(), ld, d1, k2, ll, vp, ld, dv, sv,
      own_row.data_ptr(), inv_freq.data_ptr(), sink.data_ptr(), g.data_ptr(),
      ldg, out.data_ptr(), (int)H, (int)d1, (int)d2,
      (int)(2 * inv_freq.numel()), (int)dv, (int)window, (float)scale, f32,
      stream()));
  return out;
}

// q [b, H, rank + rot] over the latent ring -> part [b, splits, H, rank + 2]
T_ attn_window_decode(T_ q, T_ ring, T_ seq, T_ cu, T_ slots, T_ lens,
                      long rank, long window, long splits, double scale,
                      bool general) {
  const SeqView sv = view(seq, cu, slots, lens);
  const bool f32 = storage(q, "q");
  check(q, q.scalar_type(), "q");
  check(ring, q.scalar_type(), "ring");
  const long H = q.size(1), D = q.size(2);
  TORCH_CHECK(sv.n == sv.b && q.size(0) == sv.b && ring.dim() == 3 &&
                  ring.size(2) == D && ring.size(0) == lens.numel() &&
                  rank <= D && window > 0 && splits > 0,
              "attn_window_decode: shape mismatch");
  auto part = torch::empty({sv.b, splits, H, rank + 2},
                           q.options().dtype(torch::kFloat32));
  if (!f32 && !general &&
      lfmq_attn_latent_decode_mfma_ok(q.data_ptr(), ring.data_ptr(), (int)rank,
                                      (int)(D - rank))) {
    CHECK_HIP(lfmq_attn_latent_decode_mfma(
        q.data_ptr(), ring.data_ptr(), sv, part.data_ptr(), (int)H, (int)rank,
        (int)(D - rank), (int)window, (int)ring.size(1), (int)splits,
        (float)scale, stream()));
    return part;
  }
  CHECK_HIP(lfmq_attn_window_decode(q.data_ptr(), ring.data_ptr(), sv,
                                    part.data_ptr(), (int)H, (int)rank,
                                    (int)(D - rank), (int)window,
                                    (int)ring.size(1), (int)splits,
                                    (float)scale, f32, stream()));
  return part;
}

bool al16(const T_& t) { return ((u64)t.data_ptr() & 15) == 0; }

// fp32 per-channel parameter of the given length
const void* vec32(const T_& t, long n, const char* name) {
  check(t, torch::kFloat32, name);
  TORCH_CHECK(t.numel() == n, name, " must have ", n, " entries");
  return t.data_ptr();
}

// {x, h}: x = rms(table[tok]) * w in fp32, h = x in the table's dtype (x
// itself in 32 bit)
std::vector<T_> embed_norm(T_ tok, T_ table, T_ w, double eps) {
  check(tok, torch::kInt64, "tok");
  const bool f32 = storage(table, "table");
  check(table, table.scalar_type(), "table");
  TORCH_CHECK(table.dim() == 2 && tok.numel() > 0, "embed_norm: shape");
  const long n = tok.numel(), width = table.size(1);
  const void* wp = vec32(w, width, "norm weight");
  auto x = torch::empty({n, width}, table.options().dtype(torch::kFloat32));
  T_ h = f32 ? x : torch::empty({n, width}, table.options());
  CHECK_HIP(lfmq_embed_norm(x.data_ptr(), table.data_ptr(), tok.data_ptr(),
                            wp, f32 ? nullptr : h.data_ptr(), (int)n,
                            (int)width, (int)table.size(0), (float)eps, f32,
                            stream()));
  return {x, h};
}

struct NormOut {
  T_ h;
  const void* w_out;
  void* hp;
};

NormOut norm_out(const T_& x, const OptT& w_out, bool f32) {
  check(x, torch::kFloat32, "x");
  TORCH_CHECK(x.dim() == 2 && x.size(0) > 0, "x must be [rows, width]");
  NormOut o;
  const bool copy = w_out.has_value() || !f32;
  o.h = copy ? torch::empty_like(x, x.options().dtype(
                                        f32 ? torch::kFloat32
                                            : torch::kBFloat16))
             : x;
  o.hp = copy ? o.h.data_ptr() : nullptr;
  o.w_out = w_out.has_value() ? vec32(*w_out, x.size(1), "output norm weight")
                              : nullptr;
  return o;
}

// x += rms(y) * w; returns x in y's dtype, or rms(x) * w_out * gain
T_ post_norm(T_ x, T_ y, T_ w, double eps, OptT w_out, double gain) {
  const bool f32 = storage(y, "y");
  check(y, y.scalar_type(), "y");
  const NormOut o = norm_out(x, w_out, f32);
  TORCH_CHECK(y.sizes() == x.sizes(), "post_norm: shape mismatch");
  CHECK_HIP(lfmq_post_norm(x.data_ptr(), y.data_ptr(),
                           vec32(w, x.size(1), "norm weight"), o.w_out, o.hp,
                           (int)x.size(0), (int)x.size(1), (float)eps,
                           (float)gain, f32, stream()));
  return o.h;
}

// the same, y the sum of rows[pos[t, :]] and sgate[t] * shared[t]
T_ post_norm_experts(T_ x, T_ rows, T_ pos, OptT shared, OptT sgate, T_ w,
                     double eps, OptT w_out, double gain) {
  const bool f32 = storage(rows, "rows");
  check(rows, rows.scalar_type(), "rows");
  check(pos, torch::kInt32, "pos");
  const NormOut o = norm_out(x, w_out, f32);
  const long n = x.size(0), width = x.size(1);
  TORCH_CHECK(rows.dim() == 2 && rows.size(1) == width && pos.dim() == 2 &&
                  pos.size(0) == n && pos.numel() == rows.size(0),
              "post_norm_experts: shape mismatch");
  const void *sh = nullptr, *sg = nullptr;
  if (shared.has_value()) {
    check(*shared, rows.scalar_type(), "shared");
    TORCH_CHECK(shared->numel() == n * width && sgate.has_value(),
                "post_norm_experts: shared expert mismatch");
    sh = shared->data_ptr();
    sg = vec32(*sgate, n, "shared gate");
  }
  CHECK_HIP(lfmq_post_norm_experts(
      x.data_ptr(), rows.data_ptr(), pos.data_ptr(), (int)pos.size(1), sh, sg,
      vec32(w, width, "norm weight"), o.w_out, o.hp, (int)n, (int)width,
      (float)eps, (float)gain, f32, stream()));
  return o.h;
}

// in rows [q | k | v]; kc [slots, cap, kv, dim], vc [slots, cap, kv, dv]
T_ qk_prep(T_ in, T_ seq, T_ cu, T_ slots, T_ lens, T_ wq, T_ wk, T_ inv_freq,
           T_ kc, T_ vc, double eps) {
  const SeqView sv = view(seq, cu, slots, lens);
  const bool f32 = storage(in, "in");
  check(kc, in.scalar_type(), "key cache");
  check(vc, in.scalar_type(), "value cache");
  check(wq, torch::kFloat32, "query norm");
  check(inv_freq, torch::kFloat32, "inv_freq");
  TORCH_CHECK(kc.dim() == 4 && vc.dim() == 4 && kc.size(0) == lens.numel() &&
                  vc.size(0) == kc.size(0) && vc.size(1) == kc.size(1) &&
                  vc.size(2) == kc.size(2),
              "qk_prep: cache mismatch");
  const long kv = kc.size(2), dim = kc.size(3), dv = vc.size(3);
  const long nq = wq.numel(), nk = kv * dim, nv = kv * dv;
  const long ld = row_stride(in, nq + nk + nv, "in"), half = inv_freq.numel();
  TORCH_CHECK(in.size(0) == sv.n && nq > 0 && nq % dim == 0 &&
                  2 * half <= dim,
              "qk_prep: shape mismatch");
  auto q = torch::empty({sv.n, nq}, in.options());
  CHECK_HIP(lfmq_qk_prep(in.data_ptr(), ld, sv, wq.data_ptr(),
                         vec32(wk, nk, "key norm"), inv_freq.data_ptr(),
                         q.data_ptr(), kc.data_ptr(), vc.data_ptr(),
                         (int)kc.size(1), (int)nq, (int)nk, (int)nv, (int)dim,
                         (int)half, (float)eps, f32, stream()));
  return q;
}

// q [N, heads * dim] ready, over the cache; writes out's columns
void attn_grouped(T_ q, T_ kc, T_ vc, T_ seq, T_ cu, T_ slots, T_ lens,
                  T_ sink, T_ out, double scale, double gain, long max_count,
                  bool general) {
  const SeqView sv = view(seq, cu, slots, lens);
  const bool f32 = storage(q, "q");
  check(q, q.scalar_type(), "q");
  check(kc, q.scalar_type(), "key cache");
  check(vc, q.scalar_type(), "value cache");
  check(sink, torch::kFloat32, "sink");
  TORCH_CHECK(kc.dim() == 4 && vc.dim() == 4 && kc.size(0) == lens.numel() &&
                  vc.size(0) == kc.size(0) && vc.size(1) == kc.size(1) &&
                  vc.size(2) == kc.size(2),
              "attn_grouped: cache mismatch");
  const long H = sink.numel(), kv = kc.size(2), dim = kc.size(3);
  const long dv = vc.size(3), cap = kc.size(1);
  const long ldo = row_stride(out, H * dv, "out");
  TORCH_CHECK(H % kv == 0 && H <= 65535 && q.numel() == sv.n * H * dim &&
                  out.size(0) == sv.n && out.scalar_type() == q.scalar_type(),
              "attn_grouped: shape mismatch");
  const int g = (int)(H / kv);
  const bool fast = !f32 && !general &&
                    lfmq_attn_grouped_mfma_ok(q.data_ptr(), kc.data_ptr(),
                                              vc.data_ptr(), (int)dim,
                                              (int)dv);
  if (fast && max_count == 1 && sv.n == sv.b) {
    const int splits = lfmq_attn_grouped_splits(sv.b, (int)H, g, (int)cap);
    T_ part;
    if (splits > 1)
      part = torch::empty({sv.b, splits, H, dv + 2},
                          q.options().dtype(torch::kFloat32));
    CHECK_HIP(lfmq_attn_grouped_decode(
        q.data_ptr(), kc.data_ptr(), vc.data_ptr(), sv, sink.data_ptr(),
        splits > 1 ? part.data_ptr() : nullptr, out.data_ptr(), ldo, (int)H,
        g, (int)dim, (int)dv, (int)cap, splits, (float)scale, (float)gain,
        stream()));
  } else if (fast) {
    CHECK_HIP(lfmq_attn_grouped_mfma(
        q.data_ptr(), kc.data_ptr(), vc.data_ptr(), sv, sink.data_ptr(),
        out.data_ptr(), ldo, (int)H, g, (int)dim, (int)dv, (int)cap,
        (float)scale, (float)gain, (int)max_count, stream()));
  } else {
    CHECK_HIP(lfmq_attn_grouped(q.data_ptr(), kc.data_ptr(), vc.data_ptr(),
                                sv, sink.data_ptr(), out.data_ptr(), ldo,
                                (int)H, g, (int)dim, (int)dv, (int)cap,
                                (float)scale, (float)gain, f32, stream()));
  }
}

// x and y: column views of one projection [N, *]; gw [blocks, 2, n, n],
// gb [blocks, 2, n]; cw [taps, C], ring [slots, taps, C], S [slots, C].  tile0 [b] first
// 64-token tile of each sequence, `tiles` in all.
void gated_lru(T_ x, T_ y, T_ seq, T_ cu, T_ slots, T_ lens, T_ xb, T_ yb,
               T_ cw, T_ cb, T_ gw, T_ gb, T_ lam, T_ ring, T_ S, T_ out,
               double c, double gain, OptT tile0, long tiles, long max_count,
               bool general) {
  const SeqView sv = view(seq, cu, slots, lens);
  const bool f32 = storage(x, "x");
  check(gw, x.scalar_type(), "gate weights");
  TORCH_CHECK(gw.dim() == 4 && gw.size(1) == 2 && gw.size(2) == gw.size(3),
              "gate weights must be [blocks, 2, n, n]");
  const long blocks = gw.size(0), n = gw.size(2), C = blocks * n;
  const long ld = row_stride(x, C, "x"), ldo = row_stride(out, C, "out");
  check(ring, torch::kFloat32, "conv ring");
  check(S, torch::kFloat32, "S");
  TORCH_CHECK(ring.dim() == 3 && ring.size(2) == C &&
                  ring.size(0) == lens.numel() &&
                  S.numel() == lens.numel() * C &&
                  row_stride(y, C, "y") == ld && x.size(0) == sv.n &&
                  y.size(0) == sv.n && out.size(0) == sv.n &&
                  y.scalar_type() == x.scalar_type() &&
                  out.scalar_type() == x.scalar_type() && blocks <= 65535,
              "gated_lru: shape mismatch");
  const long taps = ring.size(1);
  const bool mfma =
      !f32 && !general && lfmq_lru_mfma_ok(gw.data_ptr(), (int)n, (int)taps) &&
      al16(cw) && al16(cb) && al16(xb) && al16(ring);
  const bool single = sv.n == sv.b && max_count == 1;
  T_ u, ab, ends;
  if (!(mfma && single)) {
    u = torch::empty({sv.n, C}, x.options());
    ab = torch::empty({sv.n, C, 2}, S.options());
  }
  const void* t0 = nullptr;
  if (mfma && !single) {
    TORCH_CHECK(tile0.has_value() && tile0->numel() == sv.b && tiles >= sv.b,
                "gated_lru: tiles missing");
    check(*tile0, torch::kInt32, "tile0");
    t0 = tile0->data_ptr();
    ends = torch::empty({tiles, C, 2}, S.options());
  }
  auto ptr = [](const T_& t) { return t.defined() ? t.data_ptr() : nullptr; };
  CHECK_HIP(lfmq_gated_lru(
      sv, x.data_ptr(), y.data_ptr(), ld, vec32(xb, C, "x bias"),
      vec32(yb, C, "y bias"), vec32(cw, C * taps, "conv weight"),
      vec32(cb, C, "conv bias"), gw.data_ptr(), vec32(gb, 2 * C, "gate bias"),
      vec32(lam, C, "lam"), ring.data_ptr(), S.data_ptr(), out.data_ptr(),
      ldo, (int)C, (int)blocks, (int)taps, (float)c, (float)gain, ptr(u),
      ptr(ab), ptr(ends), t0, (int)max_count, single, mfma, f32, stream()));
}

// rows a tile for `pairs` (token, choice) pairs; `aligned`: the matrix-core
// products apply
long moe_tile(long pairs, long experts, bool aligned) {
  if (!aligned) return 8;
  return pairs >= 32 * experts ? 128 : 16;
}

// w [E (+ 1 with the shared expert's gate), width].  Returns {src, weight,
// pos [n, top], tiles [t, 3], shared gate [n] or empty}
std::vector<T_> moe_route(T_ h, T_ w, long E, long top, long bm) {
  const bool f32 = storage(h, "h");
  check(h, h.scalar_type(), "h");
  check(w, h.scalar_type(), "router");
  const long n = h.size(0), width = h.size(1);
  TORCH_CHECK(h.dim() == 2 && w.dim() == 2 && w.size(1) == width && n > 0 &&
                  (w.size(0) == E || w.size(0) == E + 1) && top >= 1 &&
                  top <= E && bm >= 1 && n * top < INT32_MAX,
              "moe_route: shape mismatch");
  const bool sg = w.size(0) > E;
  const long pairs = n * top;
  const long tiles = pairs / bm + (E < pairs ? E : pairs);
  auto io = h.options().dtype(torch::kInt32);
  auto fo = h.options().dtype(torch::kFloat32);
  auto ids = torch::empty({pairs}, io), src = torch::empty({pairs}, io);
  auto pos = torch::empty({n, top}, io), tl = torch::empty({tiles, 3}, io);
  auto score = torch::empty({pairs}, fo), weight = torch::empty({pairs}, fo);
  auto gate = torch::empty({sg ? n : 0}, fo);
  const bool mfma = !f32 && width % 8 == 0 && al16(h) && al16(w);
  CHECK_HIP(lfmq_moe_route_sort(
      h.data_ptr(), w.data_ptr(), ids.data_ptr(), score.data_ptr(),
      sg ? gate.data_ptr() : nullptr, src.data_ptr(), weight.data_ptr(),
      pos.data_ptr(), tl.data_ptr(), (int)n, (int)width, (int)E, (int)top,
      (int)bm, (int)tiles, mfma, f32, stream()));
  return {src, weight, pos, tl, gate};
}

// act [pairs, ff] of h's rows src, gu [E, 2 ff, width]
T_ moe_glu(T_ h, T_ gu, T_ src, T_ weight, T_ tiles, double limit,
           double alpha, double beta, long bm) {
  const bool f32 = storage(h, "h");
  check(h, h.scalar_type(), "h");
  check(gu, h.scalar_type(), "gate_up");
  check(src, torch::kInt32, "src");
  check(tiles, torch::kInt32, "tiles");
  const long pairs = src.numel(), ff = gu.size(1) / 2, K = h.size(1);
  TORCH_CHECK(gu.dim() == 3 && gu.size(2) == K && gu.size(1) == 2 * ff &&
                  (bm < 16 || (!f32 && K % 8 == 0 && al16(h) && al16(gu))),
              "moe_glu: shape mismatch");
  auto out = torch::empty({pairs, ff}, h.options());
  CHECK_HIP(lfmq_moe_glu(h.data_ptr(), gu.data_ptr(), src.data_ptr(),
                         vec32(weight, pairs, "weight"), tiles.data_ptr(),
                         out.data_ptr(), (int)ff, (int)K, (float)limit,
                         (float)alpha, (float)beta, (int)tiles.size(0),
                         (int)bm, f32, stream()));
  return out;
}

// rows [pairs, width] of act [pairs, ff], down [E, width, ff]
T_ moe_down(T_ act, T_ down, T_ tiles, long bm) {
  const bool f32 = storage(act, "act");
  check(act, act.scalar_type(), "act");
  check(down, act.scalar_type(), "down");
  check(tiles, torch::kInt32, "tiles");
  const long K = act.size(1), N = down.size(1);
  TORCH_CHECK(down.dim() == 3 && down.size(2) == K &&
                  (bm < 16 || (!f32 && K % 8 == 0 && al16(act) && al16(down))),
              "moe_down: shape mismatch");
  auto out = torch::empty({act.size(0), N}, act.options());
  CHECK_HIP(lfmq_moe_down(act.data_ptr(), down.data_ptr(), tiles.data_ptr(),
                          out.data_ptr(), (int)N, (int)K, (int)tiles.size(0),
                          (int)bm, f32, stream()));
  return out;
}

T_ clamped_glu(T_ gu, double limit, double alpha, double beta) {
  const bool f32 = storage(gu, "gate_up");
  check(gu, gu.scalar_type(), "gate_up");
  const long ff = gu.size(-1) / 2, rows = gu.numel() / gu.size(-1);
  TORCH_CHECK(gu.size(-1) == 2 * ff && rows > 0, "odd gate_up width");
  auto sizes = gu.sizes().vec();
  sizes.back() = ff;
  auto y = torch::empty(sizes, gu.options());
  CHECK_HIP(lfmq_clamped_glu(gu.data_ptr(), y.data_ptr(), rows, (int)ff,
                             (float)limit, (float)alpha, (float)beta, f32,
                             stream()));
  return y;
}

T_ silu_mul_fused(T_ gu) {
  const bool f32 = storage(gu, "gate_up");
  check(gu, gu.scalar_type(), "gate_up");
  const long inter = gu.size(-1) / 2;
  TORCH_CHECK(gu.size(-1) == 2 * inter && inter > 0, "odd gate_up width");
  const long rows = gu.numel() / (2 * inter);
  auto sizes = gu.sizes().vec();
  sizes.back() = inter;
  auto y = torch::empty(sizes, gu.options());
  if (!f32 && inter % 2 == 0)
    CHECK_HIP(lfmq_silu_mul_fused(gu.data_ptr(), y.data_ptr(), rows,
                                  (int)inter, stream()));
  else
    CHECK_HIP(lfmq_silu_mul_any(gu.data_ptr(), y.data_ptr(), rows, (int)inter,
                                f32, stream()));
  return y;
}

T_ greedy_sample(T_ logits) {
  const bool f32 = storage(logits, "logits");
  check(logits, logits.scalar_type(), "logits");
  TORCH_CHECK(logits.dim() == 2, "logits must be [b, vocab]");
  const int b = (int)logits.size(0), vocab = (int)logits.size(1);
  auto out = torch::empty({b}, logits.options().dtype(torch::kInt64));
  auto sf = torch::empty({b * 64}, logits.options().dtype(torch::kFloat32));
  auto si = torch::empty({b * 64}, logits.options().dtype(torch::kInt32));
  if (!f32 && vocab % 2 == 0)
    CHECK_HIP(lfmq_argmax_rows(logits.data_ptr(), out.data_ptr(),
                               sf.data_ptr(), si.data_ptr(), b, vocab,
                               stream()));
  else
    CHECK_HIP(lfmq_argmax_rows_any(logits.data_ptr(), out.data_ptr(),
                                   sf.data_ptr(), si.data_ptr(), b, vocab,
                                   f32, stream()));
  return out;
}

void advance_record(T_ state, T_ tok_buf, T_ sampled, T_ ring) {
  check(state, torch::kInt32, "state");
  CHECK_HIP(lfmq_advance_record(state.data_ptr(), tok_buf.data_ptr(),
                                sampled.data_ptr(), ring.data_ptr(),
                                (int)tok_buf.size(0), (int)ring.size(-1),
                                stream()));
}

}  // namespace

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.def("bigram_embed", &bigram_embed, "token + hashed bigram embedding");
  m.def("seq_advance", &seq_advance, "close a step of packed sequences");
  m.def("add_norm", &add_norm, "fp32 residual add + norm + side projection");
  m.def("head_norm_gate", &head_norm_gate, "per-head norm, weight and gate");
  m.def("mlstm_scan", &mlstm_scan, "matrix-memory recurrence, token by token");
  m.def("mlstm_chunk_ok", &mlstm_chunk_ok, "shape check of mlstm_chunk");
  m.def("mlstm_chunk", &mlstm_chunk,
        "matrix-memory recurrence by chunks, normed and gated");
  m.def("latent_prep", &latent_prep, "latent norms + shared rotated key");
  m.def("latent_ring", &latent_ring, "ring cache <-> step key buffer");
  m.def("latent_absorb", &latent_absorb, "queries into the latent space");
  m.def("latent_expand", &latent_expand, "merge, sink, values, output gate");
  m.def("attn_window_prompt", &attn_window_prompt,
        "windowed sink attention over a step's keys");
  m.def("attn_window_decode", &attn_window_decode,
        "windowed attention over the latent ring");
  m.def("embed_norm", &embed_norm, "normed embedding rows");
  m.def("post_norm", &post_norm, "norm a sublayer's output, add, cast or norm");
  m.def("post_norm_experts", &post_norm_experts,
        "sum of experts, normed, added, cast or normed");
  m.def("qk_prep", &qk_prep, "query/key norms, rotation, cache write");
  m.def("attn_grouped", &attn_grouped, "grouped-query sink attention");
  m.def("gated_lru", &gated_lru, "convolution + gated linear recurrence");
  m.def("moe_tile", &moe_tile, "rows a tile of the expert products");
  m.def("moe_route", &moe_route, "sigmoid top-k router and expert sort");
  m.def("moe_glu", &moe_glu, "gate/up products and clamped GLU");
  m.def("moe_down", &moe_down, "down products of the experts");
  m.def("clamped_glu", &clamped_glu, "clamped GLU on fused gate_up");
  m.def("silu_mul_fused", &silu_mul_fused, "silu-mul on fused gate_up");
  m.def("greedy_sample", &greedy_sample, "row argmax");
  m.def("advance_record", &advance_record, "graph decode-state advance");
}
