// Python bindings for the gfx950 kernel set (hyperspot._C).
//
// Host-side glue only — every kernel lives in a .hip translation unit and
// is reached through a plain launcher so this file needs no device code.
#include "bindings.h"

#include <array>

#include "recurrent.h"

void launch_rmsnorm(bf16*, const bf16*, const bf16*, float, long, int,
                    hipStream_t);
void launch_fused_add_rmsnorm(bf16*, bf16*, const bf16*, float, long, int,
                              hipStream_t);
void launch_rope_kv_append(bf16*, bf16*, const bf16*, const long*,
                           const float*, const long*, bf16*, bf16*, long,
                           int, int, int, int, long, long, long, bool,
                           hipStream_t);
void launch_paged_attn(bf16*, const bf16*, const bf16*, const bf16*,
                       const int*, const int*, const int*, long, int, int,
                       int, int, int, float, long, float*, int, bool,
                       hipStream_t);
void launch_attn_prefill_mfma(bf16*, const bf16*, const bf16*,
                              const bf16*, const int*, int, int, int, int,
                              int, float, long, long, long, hipStream_t);
template <typename T>
void launch_gelu_mul(T*, const T*, long, int, hipStream_t);
template <typename T>
void launch_embed_dyt(T*, float*, const T*, const long*, const float*,
                      const float*, const float*, long, int, long,
                      hipStream_t);
template <typename T>
void launch_add_dyt(T*, float*, const T*, const float*, const float*,
                    const float*, const float*, const float*, const float*,
                    long, int, hipStream_t);
template <typename T>
void launch_rope_pairs_append(T*, const T*, const T*, const long*,
                              const double*, const long*, T*, T*, long, int,
                              int, int, int, int, int, int, long, long, long,
                              hipStream_t);
template <typename T>
void launch_window_attn_general(T*, const T*, const T*, const T*, const int*,
                                const long*, const int*, const float*, long,
                                int, int, int, int, int, int, float, float,
                                float, long, hipStream_t);
void launch_window_attn_prefill(bf16*, const bf16*, const bf16*, const bf16*,
                                const int*, const long*, const int*,
                                const int*, const float*, int, int, int, int,
                                int, int, int, float, float, float, long,
                                hipStream_t);
void launch_window_attn_decode(bf16*, const bf16*, const bf16*, const bf16*,
                               const int*, const long*, const float*, float*,
                               long, int, int, int, int, int, int, float,
                               float, float, long, int, hipStream_t);
bool recurrent_chunk_fits(int, int, int);
void launch_gla_chunk_gates(float*, const bf16*, const bf16*, const float*,
                            const int*, const int*, int, int, int, float,
                            long, hipStream_t);
void launch_mlstm_chunk_gates(float*, float*, const float*, const float*,
                              const float*, const int*, const int*, int, int,
                              float, hipStream_t);
void launch_recurrent_chunk(Kind, bf16*, float*, float*, float*, float*,
                            float*, float*, float*, const bf16*, const bf16*, const bf16*,
                            const bf16*, const float*, const float*,
                            const float*, const int*, const long*,
                            const int*, const int*, const int*, int, int,
                            int, int, int, long, float, float, hipStream_t);
template <typename T>
void launch_gla_decay(float*, const T*, const T*, const float*, long, int,
                      int, float, long, hipStream_t);
void launch_mlstm_gates(float*, const float*, const float*, const float*,
                        long, int, float, hipStream_t);
template <typename T>
void launch_recurrent_scan(Kind, float*, float*, float*, float*, float*,
                           const T*, const T*, const T*, const float*, const int*,
                           const long*, const int*, int, int, int, int, long,
                           float, hipStream_t);
template <typename T>
void launch_recurrent_out(T*, const float*, const T*, const float*, bool,
                          long, int, int, long, float, hipStream_t);
template <typename T>
void launch_recurrent_step(Kind, T*, float*, float*, float*, float*,
                           const T*, const T*,
                           const T*, const T*, const T*, const T*,
                           const float*, const float*, const float*,
                           const float*, const long*, const int*, long, int,
                           int, int, int, long, float, float, float,
                           hipStream_t);
void launch_silu_mul(bf16*, const bf16*, long, int, hipStream_t);
void launch_quant_fp8(unsigned char*, float*, const bf16*, long, int, long,
                      hipStream_t);
void launch_fused_add_rmsnorm_fp8(unsigned char*, float*, const bf16*,
                                  bf16*, const bf16*, float, long, int,
                                  hipStream_t);
void launch_silu_mul_fp8(unsigned char*, float*, const bf16*, long, int,
                         hipStream_t);
void launch_moe_align(int*, int*, int*, const int*, int, int, int,
                      hipStream_t);
void launch_moe_gemm(bf16*, float*, const bf16*, const bf16*, const int*,
                     const int*, int, int, int, int, int, hipStream_t);
void launch_moe_combine(bf16*, const bf16*, const float*, const int*, long,
                        int, int, hipStream_t);
void launch_moe_gemm_fp8(bf16*, float*, const unsigned char*, const float*,
                         const unsigned char*, const float*, const int*,
                         const int*, int, int, int, int, int, hipStream_t);
template <typename T>
void launch_greedy_sample(long*, const T*, long, int, hipStream_t);
void launch_inv_cdf_sample(long*, const float*, const float*, long, int,
                           hipStream_t);

namespace {

bf16* bf(torch::Tensor& t) { return reinterpret_cast<bf16*>(t.data_ptr()); }
const bf16* cbf(const torch::Tensor& t) {
  return reinterpret_cast<const bf16*>(t.data_ptr());
}

void rmsnorm(torch::Tensor out, torch::Tensor x, torch::Tensor w,
             double eps) {
  check(out, torch::kBFloat16, "out");
  check(x, torch::kBFloat16, "x");
  check(w, torch::kBFloat16, "w");
  const int hidden = (int)x.size(-1);
  TORCH_CHECK(hidden % 8 == 0 && hidden <= 16384, "hidden size");
  launch_rmsnorm(bf(out), cbf(x), cbf(w), (float)eps, x.numel() / hidden,
                 hidden, stream());
}

void fused_add_rmsnorm(torch::Tensor x, torch::Tensor residual,
                       torch::Tensor w, double eps) {
  check(x, torch::kBFloat16, "x");
  check(residual, torch::kBFloat16, "residual");
  const int hidden = (int)x.size(-1);
  TORCH_CHECK(hidden % 8 == 0 && hidden <= 16384, "hidden size");
  launch_fused_add_rmsnorm(bf(x), bf(residual), cbf(w), (float)eps,
                           x.numel() / hidden, hidden, stream());
}

// q/k/v may be strided views into one fused qkv buffer: require only the
// head dim contiguous (stride(2)==1) and head stride == D.
void check_qkv_view(const torch::Tensor& t, const char* name) {
  TORCH_CHECK(t.is_cuda(), name, " must be on GPU");
  TORCH_CHECK(t.scalar_type() == torch::kBFloat16, name, " must be bf16");
  TORCH_CHECK(t.dim() == 3 && t.stride(2) == 1 &&
                  t.stride(1) == t.size(2),
              name, " must be [T, H, D] with contiguous heads");
}

void rope_kv_append(torch::Tensor q, torch::Tensor k, torch::Tensor v,
                    torch::Tensor positions, torch::Tensor cos_sin,
                    torch::Tensor slot_mapping, torch::Tensor k_cache,
                    torch::Tensor v_cache) {
  check_qkv_view(q, "q");
  check_qkv_view(k, "k");
  check_qkv_view(v, "v");
  check(cos_sin, torch::kFloat32, "cos_sin");
  check(positions, torch::kInt64, "positions");
  check(slot_mapping, torch::kInt64, "slot_mapping");
  const long T = q.size(0);
  const int H = (int)q.size(1), KV = (int)k.size(1), D = (int)q.size(2);
  const int BS = (int)k_cache.size(2);
  const bool kv_fp8 =
      k_cache.scalar_type() == torch::kFloat8_e4m3fn;
  launch_rope_kv_append(bf(q), bf(k), cbf(v),
                        positions.data_ptr<long>(),
                        cos_sin.data_ptr<float>(),
                        slot_mapping.data_ptr<long>(), bf(k_cache),
                        bf(v_cache), T, H, KV, D, BS, q.stride(0),
                        k.stride(0), v.stride(0), kv_fp8, stream());
}

void paged_attn(torch::Tensor out, torch::Tensor q, torch::Tensor k_cache,
                torch::Tensor v_cache, torch::Tensor block_tables,
                torch::Tensor ctx_lens,
                c10::optional<torch::Tensor> row_seq, double scale,
                c10::optional<torch::Tensor> split_ws, long split) {
  check(out, torch::kBFloat16, "out");
  check_qkv_view(q, "q");
  check(block_tables, torch::kInt32, "block_tables");
  check(ctx_lens, torch::kInt32, "ctx_lens");
  const long R = q.size(0);
  const int H = (int)q.size(1), D = (int)q.size(2);
  const int KV = (int)k_cache.size(1), BS = (int)k_cache.size(2);
  TORCH_CHECK(H % KV == 0, "GQA group");
  const int* rs = nullptr;
  if (row_seq.has_value()) {
    check(*row_seq, torch::kInt32, "row_seq");
    rs = row_seq->data_ptr<int>();
  }
  float* ws = nullptr;
  if (split > 1) {
    TORCH_CHECK(split_ws.has_value(), "split>1 needs a workspace");
    check(*split_ws, torch::kFloat, "split_ws");
    TORCH_CHECK(split_ws->numel() >= R * KV * split * (H / KV) * (D + 2),
                "split_ws too small");
    ws = split_ws->data_ptr<float>();
  }
  const bool kv_fp8 =
      k_cache.scalar_type() == torch::kFloat8_e4m3fn;
  TORCH_CHECK(v_cache.scalar_type() == k_cache.scalar_type(),
              "k/v cache dtype mismatch");
  launch_paged_attn(bf(out), cbf(q), cbf(k_cache), cbf(v_cache),
                    block_tables.data_ptr<int>(), ctx_lens.data_ptr<int>(),
                    rs, R, KV, H / KV, D, (int)block_tables.size(1), BS,
                    (float)scale, q.stride(0), ws, (int)split, kv_fp8,
                    stream());
}

void attn_prefill_mfma(torch::Tensor out, torch::Tensor q, torch::Tensor k,
                       torch::Tensor v, torch::Tensor seq_start,
                       long max_seqlen, double scale) {
  check(out, torch::kBFloat16, "out");
  check_qkv_view(q, "q");
  check_qkv_view(k, "k");
  check_qkv_view(v, "v");
  check(seq_start, torch::kInt32, "seq_start");
  const int H = (int)q.size(1), D = (int)q.size(2);
  const int KV = (int)k.size(1);
  launch_attn_prefill_mfma(
      bf(out), cbf(q), cbf(k), cbf(v), seq_start.data_ptr<int>(),
      (int)seq_start.numel() - 1, (int)max_seqlen, H, KV, D, (float)scale,
      q.stride(0), k.stride(0), v.stride(0), stream());
}

void silu_mul(torch::Tensor out, torch::Tensor x) {
  check(out, torch::kBFloat16, "out");
  check(x, torch::kBFloat16, "x");
  const int inter = (int)out.size(-1);
  TORCH_CHECK(x.size(-1) == 2 * inter && inter % 8 == 0, "shape");
  launch_silu_mul(bf(out), cbf(x), out.numel() / inter, inter, stream());
}

// ---- bf16 | float kernels ------------------------------------------------

void check_dyt(const torch::Tensor& w, const torch::Tensor& b,
               const torch::Tensor& a, long width) {
  check_param(w, width, "norm weight");
  check_param(b, width, "norm bias");
  check_param(a, 1, "norm alpha");
}

void gelu_mul(torch::Tensor out, torch::Tensor x) {
  check(out, x.scalar_type(), "out");
  check(x, x.scalar_type(), "x");
  const long inter = out.size(-1);
  TORCH_CHECK(x.size(-1) == 2 * inter &&
              x.numel() == 2 * out.numel(), "gelu_mul: shape");
  by_dtype(x, [&](auto tag) {
    using T = ELEM(tag);
    launch_gelu_mul<T>(ptr<T>(out), ptr<T>(x), out.numel() / inter,
                       (int)inter, stream());
  });
}

void embed_dyt(torch::Tensor out, torch::Tensor residual,
               torch::Tensor table, torch::Tensor ids, torch::Tensor w,
               torch::Tensor b, torch::Tensor a) {
  const long rows = ids.numel(), width = table.size(1);
  check(table, table.scalar_type(), "table");
  check(out, table.scalar_type(), "out");
  check(residual, torch::kFloat32, "residual");
  check(ids, torch::kInt64, "ids");
  check_dyt(w, b, a, width);
  TORCH_CHECK(out.numel() == rows * width &&
              residual.numel() == rows * width, "embed_dyt: shape");
  by_dtype(table, [&](auto tag) {
    using T = ELEM(tag);
    launch_embed_dyt<T>(ptr<T>(out), ptr<float>(residual), ptr<T>(table),
                        ids.data_ptr<long>(), ptr<float>(w), ptr<float>(b),
                        ptr<float>(a), rows, (int)width, table.size(0),
                        stream());
  });
}

void add_dyt(c10::optional<torch::Tensor> out, torch::Tensor residual,
             torch::Tensor h, torch::Tensor w1, torch::Tensor b1,
             torch::Tensor a1, torch::Tensor w2, torch::Tensor b2,
             torch::Tensor a2) {
  const long width = h.size(-1), rows = h.numel() / width;
  check(h, h.scalar_type(), "h");
  check(residual, torch::kFloat32, "residual");
  check_dyt(w1, b1, a1, width);
  check_dyt(w2, b2, a2, width);
  TORCH_CHECK(residual.numel() == h.numel(), "add_dyt: shape");
  if (out.has_value()) {
    check(*out, h.scalar_type(), "out");
    TORCH_CHECK(out->numel() == h.numel(), "add_dyt: shape");
  }
  by_dtype(h, [&](auto tag) {
    using T = ELEM(tag);
    launch_add_dyt<T>(out.has_value() ? ptr<T>(*out) : nullptr,
                      ptr<float>(residual), ptr<T>(h), ptr<float>(w1),
                      ptr<float>(b1), ptr<float>(a1), ptr<float>(w2),
                      ptr<float>(b2), ptr<float>(a2), rows, (int)width,
                      stream());
  });
}

// shapes of the transposed-V paged cache; returns {G, MD, E, BS}
std::array<int, 4> check_window_cache(const torch::Tensor& k_cache,
                                      const torch::Tensor& v_cache,
                                      torch::ScalarType dt) {
  check(k_cache, dt, "k_cache");
  check(v_cache, dt, "v_cache");
  TORCH_CHECK(k_cache.dim() == 4 && v_cache.dim() == 4 &&
                  k_cache.size(0) == v_cache.size(0) &&
                  k_cache.size(1) == v_cache.size(1) &&
                  k_cache.size(2) == v_cache.size(3),
              "window cache: k [NB, G, BS, 2D], v [NB, G, E, BS]");
  return {(int)k_cache.size(1), (int)k_cache.size(3),
          (int)v_cache.size(2), (int)k_cache.size(2)};
}

void rope_pairs_append(torch::Tensor q, torch::Tensor k, torch::Tensor v,
                       torch::Tensor positions, torch::Tensor freqs,
                       torch::Tensor slot_mapping, torch::Tensor k_cache,
                       torch::Tensor v_cache, long head_dim) {
  const auto dt = q.scalar_type();
  const auto [G, MD, E, BS] = check_window_cache(k_cache, v_cache, dt);
  const long rows = q.size(0), D = head_dim;
  TORCH_CHECK(q.dim() == 2 && q.size(1) % D == 0 && MD % D == 0,
              "rope_pairs_append: head_dim");
  check_rows(q, dt, rows, q.size(1), q.stride(0), "q");
  check_rows(k, dt, rows, (long)G * MD, k.stride(0), "k");
  check_rows(v, dt, rows, (long)G * E, v.stride(0), "v");
  check(positions, torch::kInt64, "positions");
  check(slot_mapping, torch::kInt64, "slot_mapping");
  check(freqs, torch::kFloat64, "freqs");
  TORCH_CHECK(positions.numel() == rows && slot_mapping.numel() == rows,
              "rope_pairs_append: rows");
  TORCH_CHECK(2 * freqs.numel() <= D && D <= 4096,
              "rope_pairs_append: rotary dimensions");
  by_dtype(q, [&](auto tag) {
    using T = ELEM(tag);
    launch_rope_pairs_append<T>(
        ptr<T>(q), ptr<T>(k), ptr<T>(v), positions.data_ptr<long>(),
        ptr<double>(freqs), slot_mapping.data_ptr<long>(), ptr<T>(k_cache),
        ptr<T>(v_cache), rows, (int)(q.size(1) / D), G * MD / (int)D, (int)D,
        G, E, 2 * (int)freqs.numel(), BS, q.stride(0), k.stride(0),
        v.stride(0), stream());
  });
}

void window_attn_general(torch::Tensor out, torch::Tensor q,
                         torch::Tensor k_cache, torch::Tensor v_cache,
                         torch::Tensor block_tables, torch::Tensor positions,
                         c10::optional<torch::Tensor> row_seq,
                         torch::Tensor lam, long window, double scale,
                         double diff, double eps) {
  const auto dt = q.scalar_type();
  const auto [G, MD, E, BS] = check_window_cache(k_cache, v_cache, dt);
  const long rows = q.size(0), D = MD / 2;
  TORCH_CHECK(BS == 16 && MD % 2 == 0 && E <= 1024 && D <= 4096 &&
              window >= 1, "window_attn: sizes");
  TORCH_CHECK(q.dim() == 2 && q.size(1) % MD == 0, "window_attn: q");
  const long H = q.size(1) / MD;
  TORCH_CHECK(H % G == 0, "window_attn: head groups");
  check_rows(q, dt, rows, H * MD, q.stride(0), "q");
  check(out, dt, "out");
  TORCH_CHECK(out.numel() == rows * H * E, "window_attn: out");
  check(block_tables, torch::kInt32, "block_tables");
  check(positions, torch::kInt64, "positions");
  TORCH_CHECK(positions.numel() == rows, "window_attn: rows");
  check_param(lam, 4 * D, "lam");
  const int* rs = nullptr;
  if (row_seq.has_value()) {
    check(*row_seq, torch::kInt32, "row_seq");
    TORCH_CHECK(row_seq->numel() == rows, "window_attn: row_seq");
    rs = row_seq->data_ptr<int>();
  } else {
    TORCH_CHECK(block_tables.size(0) >= rows, "window_attn: block_tables");
  }
  by_dtype(q, [&](auto tag) {
    using T = ELEM(tag);
    launch_window_attn_general<T>(
        ptr<T>(out), ptr<T>(q), ptr<T>(k_cache), ptr<T>(v_cache),
        block_tables.data_ptr<int>(), positions.data_ptr<long>(), rs,
        ptr<float>(lam), rows, (int)block_tables.size(1), (int)H, G, (int)D,
        E, (int)window, (float)scale, (float)diff, (float)eps, q.stride(0),
        stream());
  });
}

// 16-byte loads of q (rows and base), sizes of the padded kernels
bool window_attn_fits(torch::Tensor q, torch::Tensor k_cache,
                      torch::Tensor v_cache) {
  const long D = k_cache.size(3) / 2, E = v_cache.size(2);
  return q.scalar_type() == torch::kBFloat16 && D % 8 == 0 && E % 8 == 0 &&
         D <= 128 && E <= 256 && k_cache.size(3) == 2 * D &&
         q.stride(0) % 8 == 0 &&
         reinterpret_cast<uintptr_t>(q.data_ptr()) % 16 == 0;
}

struct WindowDims { int H, G, D, E; };

WindowDims check_window_fast(const torch::Tensor& out, const torch::Tensor& q,
                             const torch::Tensor& k_cache,
                             const torch::Tensor& v_cache,
                             const torch::Tensor& block_tables,
                             const torch::Tensor& positions,
                             const torch::Tensor& lam, long window) {
  const auto [G, MD, E, BS] =
      check_window_cache(k_cache, v_cache, torch::kBFloat16);
  TORCH_CHECK(window_attn_fits(q, k_cache, v_cache), "window_attn: sizes");
  const long rows = q.size(0);
  TORCH_CHECK(BS == 16 && window >= 1 && q.dim() == 2 &&
                  q.size(1) % ((long)MD * G) == 0, "window_attn: q");
  const int H = (int)(q.size(1) / MD);
  check_rows(q, torch::kBFloat16, rows, (long)H * MD, q.stride(0), "q");
  check(out, torch::kBFloat16, "out");
  TORCH_CHECK(out.numel() == rows * H * E, "window_attn: out");
  check(block_tables, torch::kInt32, "block_tables");
  check(positions, torch::kInt64, "positions");
  TORCH_CHECK(positions.numel() == rows, "window_attn: rows");
  check_param(lam, 2 * MD, "lam");
  return {H, G, MD / 2, E};
}

void window_attn_prefill(torch::Tensor out, torch::Tensor q,
                         torch::Tensor k_cache, torch::Tensor v_cache,
                         torch::Tensor block_tables, torch::Tensor positions,
                         torch::Tensor seq_start, torch::Tensor tiles,
                         torch::Tensor lam, long window, double scale,
                         double diff, double eps) {
  const auto d = check_window_fast(out, q, k_cache, v_cache, block_tables,
                                   positions, lam, window);
  check_tiles(tiles, seq_start, block_tables.size(0));
  launch_window_attn_prefill(
      bf(out), cbf(q), cbf(k_cache), cbf(v_cache),
      block_tables.data_ptr<int>(), positions.data_ptr<long>(),
      seq_start.data_ptr<int>(), tiles.data_ptr<int>(), ptr<float>(lam),
      (int)tiles.size(0), (int)block_tables.size(1), d.H, d.G, d.D, d.E,
      (int)window, (float)scale, (float)diff, (float)eps, q.stride(0),
      stream());
}

void window_attn_decode(torch::Tensor out, torch::Tensor q,
                        torch::Tensor k_cache, torch::Tensor v_cache,
                        torch::Tensor block_tables, torch::Tensor positions,
                        torch::Tensor lam,
                        c10::optional<torch::Tensor> partial, long split,
                        long window, double scale, double diff, double eps) {
  const auto d = check_window_fast(out, q, k_cache, v_cache, block_tables,
                                   positions, lam, window);
  const long rows = q.size(0);
  TORCH_CHECK(block_tables.size(0) >= rows && split >= 1 && split <= 64,
              "window_attn_decode: rows, split");
  if (split > 1) {
    TORCH_CHECK(partial.has_value(), "window_attn_decode: partial");
    check_param(*partial, rows * d.H * split * 2 * (d.E + 2), "partial");
  }
  launch_window_attn_decode(
      bf(out), cbf(q), cbf(k_cache), cbf(v_cache),
      block_tables.data_ptr<int>(), positions.data_ptr<long>(),
      ptr<float>(lam), split > 1 ? ptr<float>(*partial) : nullptr, rows,
      (int)block_tables.size(1), d.H, d.G, d.D, d.E, (int)window,
      (float)scale, (float)diff, (float)eps, q.stride(0), (int)split,
      stream());
}

void gla_decay(torch::Tensor log_decay, torch::Tensor a1h, torch::Tensor a2,
               torch::Tensor a2b, double tau) {
  const auto dt = a1h.scalar_type();
  const long rows = a1h.size(0), C = a2.size(0), R = a2.size(1);
  check_rows(a1h, dt, rows, R, a1h.stride(0), "a1h");
  check(a2, dt, "a2");
  check_param(a2b, C, "a2 bias");
  check_param(log_decay, rows * C, "log_decay");
  by_dtype(a1h, [&](auto tag) {
    using T = ELEM(tag);
    launch_gla_decay<T>(ptr<float>(log_decay), ptr<T>(a1h), ptr<T>(a2),
                        ptr<float>(a2b), rows, (int)C, (int)R, (float)tau,
                        a1h.stride(0), stream());
  });
}

void mlstm_gates(torch::Tensor out, torch::Tensor raw, torch::Tensor ib,
                 torch::Tensor fb, double cap) {
  const long H = ib.numel(), rows = raw.size(0);
  check_param(raw, rows * 2 * H, "raw gates");
  check_param(out, rows * 2 * H, "gates");
  check_param(ib, H, "input gate bias");
  check_param(fb, H, "forget gate bias");
  launch_mlstm_gates(ptr<float>(out), ptr<float>(raw), ptr<float>(ib),
                     ptr<float>(fb), rows, (int)H, (float)cap, stream());
}

struct StateDims { long slots, H, D, E; };

// S [slots, H, D, E]; n [slots, H, D] and m [slots, H] come together
StateDims check_state(const torch::Tensor& S,
                      const c10::optional<torch::Tensor>& n,
                      const c10::optional<torch::Tensor>& m) {
  check(S, torch::kFloat32, "state");
  TORCH_CHECK(S.dim() == 4 && S.size(2) <= 1024 && S.size(3) <= 1024,
              "state must be [slots, H, D <= 1024, E <= 1024]");
  TORCH_CHECK(n.has_value() == m.has_value(), "state: n and m");
  if (n.has_value()) {
    check_param(*n, S.size(0) * S.size(1) * S.size(2), "state n");
    check_param(*m, S.size(0) * S.size(1), "state m");
  }
  return {S.size(0), S.size(1), S.size(2), S.size(3)};
}

void recurrent_scan(torch::Tensor o, torch::Tensor S,
                    c10::optional<torch::Tensor> n,
                    c10::optional<torch::Tensor> m,
                    c10::optional<torch::Tensor> nm_new, torch::Tensor q,
                    torch::Tensor k, torch::Tensor v, torch::Tensor gates,
                    torch::Tensor seq_start, torch::Tensor positions,
                    torch::Tensor slots, double qscale) {
  const auto dt = q.scalar_type();
  const auto d = check_state(S, n, m);
  const long rows = q.size(0), B = slots.numel(), st = q.stride(0);
  check_rows(q, dt, rows, d.H * d.D, st, "q");
  check_rows(k, dt, rows, d.H * d.D, st, "k");
  check_rows(v, dt, rows, d.H * d.E, st, "v");
  check_param(o, rows * d.H * d.E, "o");
  check_param(gates, rows * d.H * (n.has_value() ? 2 : d.D), "gates");
  check(seq_start, torch::kInt32, "seq_start");
  check(positions, torch::kInt64, "positions");
  check(slots, torch::kInt32, "slots");
  TORCH_CHECK(seq_start.numel() == B + 1 && positions.numel() == rows &&
              B <= 65535, "recurrent_scan: sequences");
  if (n.has_value()) {
    TORCH_CHECK(nm_new.has_value(), "recurrent_scan: nm_new");
    check_param(*nm_new, B * d.H * (d.D + 1), "nm_new");
  }
  by_dtype(q, [&](auto tag) {
    using T = ELEM(tag);
    launch_recurrent_scan<T>(
        n.has_value() ? MLSTM : GLA, ptr<float>(o), ptr<float>(S), opt(n),
        opt(m), opt(nm_new), ptr<T>(q),
        ptr<T>(k), ptr<T>(v), ptr<float>(gates), seq_start.data_ptr<int>(),
        positions.data_ptr<long>(), slots.data_ptr<int>(), (int)B, (int)d.H,
        (int)d.D, (int)d.E, st, (float)qscale, stream());
  });
}

void gla_chunk_gates(torch::Tensor b, torch::Tensor a1h, torch::Tensor a2,
                     torch::Tensor a2b, torch::Tensor seq_start,
                     torch::Tensor tiles, double tau) {
  const long rows = a1h.size(0), Cn = a2.size(0), R = a2.size(1);
  check_rows(a1h, torch::kBFloat16, rows, R, a1h.stride(0), "a1h");
  check(a2, torch::kBFloat16, "a2");
  check_param(a2b, Cn, "a2 bias");
  check_param(b, rows * Cn, "b");
  check_tiles(tiles, seq_start, seq_start.numel() - 1);
  launch_gla_chunk_gates(ptr<float>(b), cbf(a1h), cbf(a2), ptr<float>(a2b),
                         seq_start.data_ptr<int>(), tiles.data_ptr<int>(),
                         (int)tiles.size(0), (int)Cn, (int)R, (float)tau,
                         a1h.stride(0), stream());
}

void mlstm_chunk_gates(torch::Tensor gates, torch::Tensor info,
                       torch::Tensor raw, torch::Tensor ib, torch::Tensor fb,
                       torch::Tensor seq_start, torch::Tensor tiles,
                       double cap) {
  const long H = ib.numel(), rows = raw.size(0);
  check_param(raw, rows * 2 * H, "raw gates");
  check_param(gates, rows * 2 * H, "gates");
  check_param(ib, H, "input gate bias");
  check_param(fb, H, "forget gate bias");
  check_tiles(tiles, seq_start, seq_start.numel() - 1);
  check_param(info, tiles.size(0) * H * 2, "info");
  launch_mlstm_chunk_gates(ptr<float>(gates), ptr<float>(info),
                           ptr<float>(raw), ptr<float>(ib), ptr<float>(fb),
                           seq_start.data_ptr<int>(), tiles.data_ptr<int>(),
                           (int)tiles.size(0), (int)H, (float)cap, stream());
}

// 16-byte loads of q, k, v, g and float4 rows of the states
bool chunk_fits(torch::Tensor S, torch::Tensor q, torch::Tensor k,
                torch::Tensor v, torch::Tensor g, long rank) {
  auto aligned = [](const torch::Tensor& t) {
    return t.scalar_type() == torch::kBFloat16 && t.stride(0) % 8 == 0 &&
           reinterpret_cast<uintptr_t>(t.data_ptr()) % 16 == 0;
  };
  return aligned(q) && aligned(k) && aligned(v) && aligned(g) &&
         recurrent_chunk_fits((int)S.size(2), (int)S.size(3), (int)rank);
}

void recurrent_chunk(torch::Tensor y, torch::Tensor U,
                     c10::optional<torch::Tensor> nU,
                     c10::optional<torch::Tensor> m_in, torch::Tensor S,
                     c10::optional<torch::Tensor> n,
                     c10::optional<torch::Tensor> m, torch::Tensor q,
                     torch::Tensor k, torch::Tensor v, torch::Tensor g,
                     torch::Tensor gates, c10::optional<torch::Tensor> info,
                     torch::Tensor w, torch::Tensor seq_start,
                     torch::Tensor positions, torch::Tensor slots,
                     torch::Tensor tiles, torch::Tensor tile_start,
                     double qscale, double eps) {
  const auto d = check_state(S, n, m);
  const auto dt = torch::kBFloat16;
  const long rows = q.size(0), st = q.stride(0), B = slots.numel();
  const bool mlstm = n.has_value();
  TORCH_CHECK(chunk_fits(S, q, k, v, g, 1), "recurrent_chunk: sizes");
  check_rows(q, dt, rows, d.H * d.D, st, "q");
  check_rows(k, dt, rows, d.H * d.D, st, "k");
  check_rows(v, dt, rows, d.H * d.E, st, "v");
  check_rows(g, dt, rows, d.H * d.E, st, "g");
  check(y, dt, "y");
  TORCH_CHECK(y.numel() == rows * d.H * d.E, "recurrent_chunk: y");
  check(positions, torch::kInt64, "positions");
  check(slots, torch::kInt32, "slots");
  check(tile_start, torch::kInt32, "tile_start");
  check_tiles(tiles, seq_start, B);
  const long nt = tiles.size(0);
  TORCH_CHECK(positions.numel() == rows && tile_start.numel() == B + 1 &&
                  B <= 65535, "recurrent_chunk: sequences");
  check_param(U, nt * d.H * d.D * d.E, "U");
  check_param(gates, rows * d.H * (mlstm ? 2 : d.D), "gates");
  check_param(w, mlstm ? d.H * d.E : d.E, "norm weight");
  if (mlstm) {
    TORCH_CHECK(nU.has_value() && m_in.has_value() && info.has_value(),
                "recurrent_chunk: scratch");
    check_param(*nU, nt * d.H * d.D, "nU");
    check_param(*m_in, nt * d.H, "m_in");
    check_param(*info, nt * d.H * 2, "info");
  }
  launch_recurrent_chunk(
      mlstm ? MLSTM : GLA, bf(y), nullptr, ptr<float>(U), opt(nU),
      opt(m_in), ptr<float>(S), opt(n),
      opt(m), cbf(q), cbf(k), cbf(v), cbf(g), ptr<float>(gates), opt(info),
      ptr<float>(w), seq_start.data_ptr<int>(), positions.data_ptr<long>(),
      slots.data_ptr<int>(), tiles.data_ptr<int>(),
      tile_start.data_ptr<int>(), (int)nt, (int)B, (int)d.H, (int)d.D,
      (int)d.E, st, (float)qscale, (float)eps, stream());
}

void recurrent_out(torch::Tensor y, torch::Tensor o, torch::Tensor g,
                   torch::Tensor w, long heads, bool mlstm, double eps) {
  const auto dt = y.scalar_type();
  const long rows = g.size(0), HE = g.size(1), E = HE / heads;
  TORCH_CHECK(HE % heads == 0, "recurrent_out: heads");
  check(y, dt, "y");
  TORCH_CHECK(y.numel() == rows * HE, "recurrent_out: y");
  check_param(o, rows * HE, "o");
  check_rows(g, dt, rows, HE, g.stride(0), "g");
  check_param(w, mlstm ? HE : E, "norm weight");
  by_dtype(y, [&](auto tag) {
    using T = ELEM(tag);
    launch_recurrent_out<T>(ptr<T>(y), ptr<float>(o), ptr<T>(g),
                            ptr<float>(w), mlstm, rows, (int)heads, (int)E,
                            g.stride(0), (float)eps, stream());
  });
}

void check_step(const torch::Tensor& y, const StateDims& d,
                const torch::Tensor& q, const torch::Tensor& k,
                const torch::Tensor& v, const torch::Tensor& g,
                const torch::Tensor& positions, const torch::Tensor& slots) {
  const auto dt = q.scalar_type();
  const long rows = q.size(0), st = q.stride(0);
  check(y, dt, "y");
  TORCH_CHECK(y.numel() == rows * d.H * d.E, "recurrent_step: y");
  check_rows(q, dt, rows, d.H * d.D, st, "q");
  check_rows(k, dt, rows, d.H * d.D, st, "k");
  check_rows(v, dt, rows, d.H * d.E, st, "v");
  check_rows(g, dt, rows, d.H * d.E, st, "g");
  check(positions, torch::kInt64, "positions");
  check(slots, torch::kInt32, "slots");
  TORCH_CHECK(positions.numel() == rows && slots.numel() == rows,
              "recurrent_step: rows");
}

void gla_step(torch::Tensor y, torch::Tensor S, torch::Tensor q,
              torch::Tensor k, torch::Tensor v, torch::Tensor g,
              torch::Tensor a1h, torch::Tensor a2, torch::Tensor a2b,
              torch::Tensor w, torch::Tensor positions, torch::Tensor slots,
              double qscale, double tau, double eps) {
  const auto d = check_state(S, c10::nullopt, c10::nullopt);
  check_step(y, d, q, k, v, g, positions, slots);
  const long rows = q.size(0), R = a2.size(1);
  check_rows(a1h, q.scalar_type(), rows, R, q.stride(0), "a1h");
  check(a2, q.scalar_type(), "a2");
  TORCH_CHECK(a2.size(0) == d.H * d.D, "gla_step: a2");
  check_param(a2b, d.H * d.D, "a2 bias");
  check_param(w, d.E, "norm weight");
  by_dtype(q, [&](auto tag) {
    using T = ELEM(tag);
    launch_recurrent_step<T>(
        GLA, ptr<T>(y), nullptr, ptr<float>(S), nullptr, nullptr, ptr<T>(q),
        ptr<T>(k),
        ptr<T>(v), ptr<T>(g), ptr<T>(a1h), ptr<T>(a2), ptr<float>(a2b),
        nullptr, nullptr, ptr<float>(w), positions.data_ptr<long>(),
        slots.data_ptr<int>(), rows, (int)d.H, (int)d.D, (int)d.E, (int)R,
        q.stride(0), (float)qscale, (float)tau, (float)eps, stream());
  });
}

void mlstm_step(torch::Tensor y, torch::Tensor S, torch::Tensor n,
                torch::Tensor m, torch::Tensor q, torch::Tensor k,
                torch::Tensor v, torch::Tensor g, torch::Tensor raw,
                torch::Tensor ib, torch::Tensor fb, torch::Tensor w,
                torch::Tensor positions, torch::Tensor slots, double qscale,
                double cap, double eps) {
  const auto d = check_state(S, n, m);
  check_step(y, d, q, k, v, g, positions, slots);
  const long rows = q.size(0);
  check_param(raw, rows * 2 * d.H, "raw gates");
  check_param(ib, d.H, "input gate bias");
  check_param(fb, d.H, "forget gate bias");
  check_param(w, d.H * d.E, "norm weight");
  by_dtype(q, [&](auto tag) {
    using T = ELEM(tag);
    launch_recurrent_step<T>(
        MLSTM, ptr<T>(y), nullptr, ptr<float>(S), ptr<float>(n),
        ptr<float>(m), ptr<T>(q),
        ptr<T>(k), ptr<T>(v), ptr<T>(g), nullptr, nullptr, ptr<float>(ib),
        ptr<float>(fb), ptr<float>(raw), ptr<float>(w),
        positions.data_ptr<long>(), slots.data_ptr<int>(), rows, (int)d.H,
        (int)d.D, (int)d.E, 0, q.stride(0), (float)qscale, (float)cap,
        (float)eps, stream());
  });
}

// q, k, v rows of one buffer, o [T, H * E] float, one decay per head
StateDims check_lightning(const torch::Tensor& o, const torch::Tensor& S,
                          const torch::Tensor& q, const torch::Tensor& k,
                          const torch::Tensor& v, const torch::Tensor& decay,
                          const torch::Tensor& positions,
                          const torch::Tensor& slots) {
  const auto d = check_state(S, c10::nullopt, c10::nullopt);
  const auto dt = q.scalar_type();
  const long rows = q.size(0), st = q.stride(0);
  check_rows(q, dt, rows, d.H * d.D, st, "q");
  check_rows(k, dt, rows, d.H * d.D, st, "k");
  check_rows(v, dt, rows, d.H * d.E, st, "v");
  check_param(o, rows * d.H * d.E, "o");
  check_param(decay, d.H, "decay");
  check(positions, torch::kInt64, "positions");
  check(slots, torch::kInt32, "slots");
  TORCH_CHECK(positions.numel() == rows, "lightning: rows");
  return d;
}

void lightning_step(torch::Tensor o, torch::Tensor S, torch::Tensor q,
                    torch::Tensor k, torch::Tensor v, torch::Tensor decay,
                    torch::Tensor positions, torch::Tensor slots) {
  const auto d = check_lightning(o, S, q, k, v, decay, positions, slots);
  TORCH_CHECK(slots.numel() == q.size(0), "lightning_step: slots");
  by_dtype(q, [&](auto tag) {
    using T = ELEM(tag);
    launch_recurrent_step<T>(
        LIGHTNING, nullptr, ptr<float>(o), ptr<float>(S), nullptr, nullptr,
        ptr<T>(q), ptr<T>(k), ptr<T>(v), nullptr, nullptr, nullptr,
        ptr<float>(decay), nullptr, nullptr, nullptr,
        positions.data_ptr<long>(), slots.data_ptr<int>(), q.size(0),
        (int)d.H, (int)d.D, (int)d.E, 0, q.stride(0), 1.f, 0.f, 0.f,
        stream());
  });
}

void lightning_scan(torch::Tensor o, torch::Tensor S, torch::Tensor q,
                    torch::Tensor k, torch::Tensor v, torch::Tensor decay,
                    torch::Tensor seq_start, torch::Tensor positions,
                    torch::Tensor slots) {
  const auto d = check_lightning(o, S, q, k, v, decay, positions, slots);
  const long B = slots.numel();
  check(seq_start, torch::kInt32, "seq_start");
  TORCH_CHECK(seq_start.numel() == B + 1 && B <= 65535,
              "lightning_scan: sequences");
  by_dtype(q, [&](auto tag) {
    using T = ELEM(tag);
    launch_recurrent_scan<T>(
        LIGHTNING, ptr<float>(o), ptr<float>(S), nullptr, nullptr, nullptr,
        ptr<T>(q), ptr<T>(k), ptr<T>(v), ptr<float>(decay),
        seq_start.data_ptr<int>(), positions.data_ptr<long>(),
        slots.data_ptr<int>(), (int)B, (int)d.H, (int)d.D, (int)d.E,
        q.stride(0), 1.f, stream());
  });
}

void lightning_chunk(torch::Tensor o, torch::Tensor U, torch::Tensor S,
                     torch::Tensor q, torch::Tensor k, torch::Tensor v,
                     torch::Tensor decay, torch::Tensor seq_start,
                     torch::Tensor positions, torch::Tensor slots,
                     torch::Tensor tiles, torch::Tensor tile_start) {
  const auto d = check_lightning(o, S, q, k, v, decay, positions, slots);
  const long B = slots.numel(), nt = tiles.size(0);
  TORCH_CHECK(chunk_fits(S, q, k, v, v, 0), "lightning_chunk: sizes");
  check(tile_start, torch::kInt32, "tile_start");
  check_tiles(tiles, seq_start, B);
  TORCH_CHECK(tile_start.numel() == B + 1 && B <= 65535,
              "lightning_chunk: sequences");
  check_param(U, nt * d.H * d.D * d.E, "U");
  launch_recurrent_chunk(
      LIGHTNING, nullptr, ptr<float>(o), ptr<float>(U), nullptr, nullptr,
      ptr<float>(S), nullptr, nullptr, ptr<bf16>(q), ptr<bf16>(k),
      ptr<bf16>(v), nullptr, ptr<float>(decay), nullptr, nullptr,
      seq_start.data_ptr<int>(), positions.data_ptr<long>(),
      slots.data_ptr<int>(), tiles.data_ptr<int>(),
      tile_start.data_ptr<int>(), (int)nt, (int)B, (int)d.H, (int)d.D,
      (int)d.E, q.stride(0), 1.f, 0.f, stream());
}

void greedy_sample(torch::Tensor out, torch::Tensor logits) {
  check(out, torch::kInt64, "out");
  if (logits.scalar_type() == torch::kFloat32) {
    check(logits, torch::kFloat32, "logits");
    launch_greedy_sample(out.data_ptr<long>(), logits.data_ptr<float>(),
                         logits.size(0), (int)logits.size(1), stream());
    return;
  }
  check(logits, torch::kBFloat16, "logits");
  launch_greedy_sample(out.data_ptr<long>(), cbf(logits), logits.size(0),
                       (int)logits.size(1), stream());
}

void inv_cdf_sample(torch::Tensor out, torch::Tensor logits,
                    torch::Tensor uniform) {
  check(out, torch::kInt64, "out");
  check(logits, torch::kFloat32, "logits");
  check(uniform, torch::kFloat32, "uniform");
  launch_inv_cdf_sample(out.data_ptr<long>(), logits.data_ptr<float>(),
                        uniform.data_ptr<float>(), logits.size(0),
                        (int)logits.size(1), stream());
}

}  // namespace


unsigned char* u8(torch::Tensor& t) {
  return reinterpret_cast<unsigned char*>(t.data_ptr());
}

void quant_fp8(torch::Tensor out, torch::Tensor scales, torch::Tensor x) {
  check(out, torch::kFloat8_e4m3fn, "out");
  check(scales, torch::kFloat, "scales");
  TORCH_CHECK(x.is_cuda() && x.scalar_type() == torch::kBFloat16, "x");
  const int hidden = (int)x.size(-1);
  TORCH_CHECK(x.stride(-1) == 1, "x inner dim must be contiguous");
  const long rows = x.numel() / hidden;
  const long stride = x.dim() > 1 ? x.stride(0) : hidden;
  launch_quant_fp8(u8(out), scales.data_ptr<float>(), cbf(x), rows, hidden,
                   stride, stream());
}

void fused_add_rmsnorm_fp8(torch::Tensor out, torch::Tensor scales,
                           torch::Tensor x, torch::Tensor residual,
                           torch::Tensor w, double eps) {
  check(out, torch::kFloat8_e4m3fn, "out");
  check(scales, torch::kFloat, "scales");
  check(x, torch::kBFloat16, "x");
  check(residual, torch::kBFloat16, "residual");
  check(w, torch::kBFloat16, "w");
  const int hidden = (int)x.size(-1);
  launch_fused_add_rmsnorm_fp8(u8(out), scales.data_ptr<float>(), cbf(x),
                               bf(residual), cbf(w), (float)eps,
                               x.numel() / hidden, hidden, stream());
}

void silu_mul_fp8(torch::Tensor out, torch::Tensor scales, torch::Tensor x) {
  check(out, torch::kFloat8_e4m3fn, "out");
  check(scales, torch::kFloat, "scales");
  check(x, torch::kBFloat16, "x");
  const int inter = (int)out.size(-1);
  TORCH_CHECK(x.size(-1) == 2 * inter, "x must be [rows, 2*inter]");
  launch_silu_mul_fp8(u8(out), scales.data_ptr<float>(), cbf(x),
                      out.numel() / inter, inter, stream());
}


void moe_align(torch::Tensor sorted_ids, torch::Tensor tile_expert,
               torch::Tensor inv_pos, torch::Tensor flat_ids,
               long num_experts) {
  check(sorted_ids, torch::kInt, "sorted_ids");
  check(tile_expert, torch::kInt, "tile_expert");
  check(inv_pos, torch::kInt, "inv_pos");
  check(flat_ids, torch::kInt, "flat_ids");
  launch_moe_align(sorted_ids.data_ptr<int>(), tile_expert.data_ptr<int>(),
                   inv_pos.data_ptr<int>(), flat_ids.data_ptr<int>(),
                   (int)flat_ids.numel(), (int)num_experts,
                   (int)tile_expert.numel(), stream());
}

void moe_gemm(torch::Tensor out, torch::Tensor x, torch::Tensor w,
              torch::Tensor sorted_ids, torch::Tensor tile_expert,
              long gather_div, long splitk,
              c10::optional<torch::Tensor> ws) {
  check(out, torch::kBFloat16, "out");
  check(x, torch::kBFloat16, "x");
  check(w, torch::kBFloat16, "w");
  check(sorted_ids, torch::kInt, "sorted_ids");
  check(tile_expert, torch::kInt, "tile_expert");
  TORCH_CHECK(w.dim() == 3, "w must be [E, N, K]");
  float* wsp = nullptr;
  if (splitk > 1) {
    TORCH_CHECK(ws.has_value(), "moe_gemm: splitk>1 needs a workspace");
    check(*ws, torch::kFloat, "ws");
    TORCH_CHECK(ws->numel() >= splitk * out.numel(),
                "moe_gemm: workspace too small");
    wsp = ws->data_ptr<float>();
  }
  launch_moe_gemm(bf(out), wsp, cbf(x), cbf(w),
                  sorted_ids.data_ptr<int>(),
                  tile_expert.data_ptr<int>(), (int)tile_expert.numel(),
                  (int)w.size(1), (int)w.size(2), (int)gather_div,
                  (int)splitk, stream());
}

void moe_combine(torch::Tensor out, torch::Tensor y, torch::Tensor wts,
                 torch::Tensor inv_pos, long topk) {
  check(out, torch::kBFloat16, "out");
  check(y, torch::kBFloat16, "y");
  check(wts, torch::kFloat, "wts");
  check(inv_pos, torch::kInt, "inv_pos");
  launch_moe_combine(bf(out), cbf(y), wts.data_ptr<float>(),
                     inv_pos.data_ptr<int>(), out.size(0), (int)topk,
                     (int)out.size(-1), stream());
}


void moe_gemm_fp8(torch::Tensor out, torch::Tensor xq, torch::Tensor xs,
                  torch::Tensor wq, torch::Tensor ws,
                  torch::Tensor sorted_ids, torch::Tensor tile_expert,
                  long gather_div, long splitk,
                  c10::optional<torch::Tensor> skw) {
  check(out, torch::kBFloat16, "out");
  check(xq, torch::kFloat8_e4m3fn, "xq");
  check(xs, torch::kFloat, "xs");
  check(wq, torch::kFloat8_e4m3fn, "wq");
  check(ws, torch::kFloat, "ws");
  check(sorted_ids, torch::kInt, "sorted_ids");
  check(tile_expert, torch::kInt, "tile_expert");
  TORCH_CHECK(wq.dim() == 3, "wq must be [E, N, K]");
  float* skp = nullptr;
  if (splitk > 1) {
    TORCH_CHECK(skw.has_value(),
                "moe_gemm_fp8: splitk>1 needs a workspace");
    check(*skw, torch::kFloat, "skw");
    TORCH_CHECK(skw->numel() >= splitk * out.numel(),
                "moe_gemm_fp8: workspace too small");
    skp = skw->data_ptr<float>();
  }
  launch_moe_gemm_fp8(bf(out), skp, u8(xq), xs.data_ptr<float>(), u8(wq),
                      ws.data_ptr<float>(), sorted_ids.data_ptr<int>(),
                      tile_expert.data_ptr<int>(),
                      (int)tile_expert.numel(), (int)wq.size(1),
                      (int)wq.size(2), (int)gather_div, (int)splitk,
                      stream());
}

void register_latent(pybind11::module_& m);    // bindings_latent.cpp
void register_sublayer(pybind11::module_& m);  // bindings_sublayer.cpp

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.doc() = "HyperSpot-AMD gfx950 (CDNA4) kernels";
  m.def("rmsnorm", &rmsnorm);
  m.def("quant_fp8", &quant_fp8);
  m.def("fused_add_rmsnorm_fp8", &fused_add_rmsnorm_fp8);
  m.def("silu_mul_fp8", &silu_mul_fp8);
  m.def("moe_align", &moe_align);
  m.def("moe_gemm", &moe_gemm);
  m.def("moe_combine", &moe_combine);
  m.def("moe_gemm_fp8", &moe_gemm_fp8);
  m.def("fused_add_rmsnorm", &fused_add_rmsnorm);
  m.def("rope_kv_append", &rope_kv_append);
  m.def("paged_attn", &paged_attn);
  m.def("attn_prefill_mfma", &attn_prefill_mfma);
  m.def("silu_mul", &silu_mul);
  m.def("gelu_mul", &gelu_mul);
  m.def("embed_dyt", &embed_dyt);
  m.def("add_dyt", &add_dyt);
  m.def("rope_pairs_append", &rope_pairs_append);
  m.def("window_attn_general", &window_attn_general);
  m.def("window_attn_fits", &window_attn_fits);
  m.def("window_attn_prefill", &window_attn_prefill);
  m.def("window_attn_decode", &window_attn_decode);
  m.def("gla_chunk_gates", &gla_chunk_gates);
  m.def("mlstm_chunk_gates", &mlstm_chunk_gates);
  m.def("chunk_fits", &chunk_fits);
  m.def("recurrent_chunk", &recurrent_chunk);
  m.def("gla_decay", &gla_decay);
  m.def("mlstm_gates", &mlstm_gates);
  m.def("recurrent_scan", &recurrent_scan);
  m.def("recurrent_out", &recurrent_out);
  m.def("gla_step", &gla_step);
  m.def("mlstm_step", &mlstm_step);
  m.def("lightning_step", &lightning_step);
  m.def("lightning_scan", &lightning_scan);
  m.def("lightning_chunk", &lightning_chunk);
  register_latent(m);
  register_sublayer(m);
  m.def("greedy_sample", &greedy_sample);
  m.def("inv_cdf_sample", &inv_cdf_sample);
}
