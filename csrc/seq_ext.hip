// lfmq_seq — torch bindings of the sequence-mixing layers' kernels (packed
// variable-length batches, recurrent states, windowed latent attention)
// and of the small ops every model shares.  Every entry checks dtypes,
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
  m.def("silu_mul_fused", &silu_mul_fused, "silu-mul on fused gate_up");
  m.def("greedy_sample", &greedy_sample, "row argmax");
  m.def("advance_record", &advance_record, "graph decode-state advance");
}
