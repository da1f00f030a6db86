// Bindings of the RMS-normed residual, latent attention and expert kernels
// (rms.hip, attn_latent.hip, experts.hip).
#include "bindings.h"

template <typename T>
void launch_embed_scaled(T*, float*, const T*, const long*, float, long, int,
                         long, hipStream_t);
template <typename T>
void launch_rms_scale(T*, const float*, const float*, long, int, float,
                      hipStream_t);
template <typename T>
void launch_add_rms(T*, float*, const T*, const float*, long, int, float,
                    hipStream_t);
template <typename T>
void launch_rms_gate(T*, const float*, const T*, const float*, const float*,
                     long, int, long, long, float, hipStream_t);
void launch_row_squares(float*, const float*, long, int, hipStream_t);
template <typename T>
void launch_gelu_gate(T*, const T*, const T*, const long*, long, int, long,
                      long, long, hipStream_t);
bool latent_sizes_fit(int, int, int, int);
template <typename T>
void launch_latent_rope_append(T*, const T*, const float*, const long*,
                               const double*, const long*, T*, long, int, int,
                               int, int, long, long, float, float,
                               const SideRelu<T>&, hipStream_t);
void launch_latent_gather(bf16*, const bf16*, const long*, long, int,
                          hipStream_t);
template <typename T>
void launch_head_gemm(T*, const T*, const T*, const int*, const int*, long,
                      int, int, int, long, long, long, long, long, long,
                      const T*, long, bool, hipStream_t);
template <typename T>
void launch_latent_attn_general(T*, const T*, const T*, const T*, const int*,
                                const long*, const int*, const int*,
                                const float*, long, int, int, int, int, int,
                                int, float, long, hipStream_t);
void launch_latent_attn_decode(bf16*, float*, const bf16*, const bf16*,
                               const bf16*, const int*, const long*,
                               const int*, const int*, const float*, long,
                               int, int, int, int, int, int, float, long, int,
                               hipStream_t);
void launch_latent_merge_values(bf16*, const float*, const bf16*, const int*,
                                long, int, int, int, int, long, const bf16*,
                                long, hipStream_t);
void launch_latent_attn_prefill(bf16*, const bf16*, const bf16*, const bf16*,
                                const bf16*, const long*, const int*,
                                const int*, const int*, const int*,
                                const float*, int, int, int, int, int, int,
                                long, int, float, long, long, const bf16*,
                                long, hipStream_t);
void launch_experts_route(float*, int*, const float*, int, int, int, bool,
                          bool, int, const float*, hipStream_t);
void launch_experts_sort(int*, int*, int*, const int*, int, int, int, int,
                         hipStream_t);
void launch_experts_route_sort(float*, int*, int*, int*, int*, const float*,
                               int, int, int, bool, int, int, int,
                               const float*, hipStream_t);
template <typename T>
void launch_experts_gemm(bool, T*, const T*, const T*, const T*, const int*,
                         const int*, int, int, int, int, int, int, int, long,
                         long, int, bool, float, hipStream_t);
template <typename T>
void launch_experts_sum(T*, float*, const T*, const T*, const T*,
                        const float*, const int*, const float*, long, int,
                        int, float, hipStream_t);

namespace {

using torch::Tensor;
using Maybe = c10::optional<Tensor>;

void check_ints(const Tensor& t, long numel, const char* name) {
  check(t, torch::kInt32, name);
  TORCH_CHECK(t.numel() == numel, name, " must have ", numel, " elements");
}

const int* opt_int(const Maybe& t) {
  return t.has_value() ? t->data_ptr<int>() : nullptr;
}

bool aligned16(const Tensor& t) {
  return reinterpret_cast<uintptr_t>(t.data_ptr()) % 16 == 0;
}

// ---- residual -------------------------------------------------------------

void embed_scaled(Maybe out, Tensor residual, Tensor table, Tensor ids,
                  double scale) {
  const long rows = ids.numel(), width = table.size(1);
  check(table, table.scalar_type(), "table");
  check(ids, torch::kInt64, "ids");
  check_param(residual, rows * width, "residual");
  if (out.has_value()) {
    check(*out, table.scalar_type(), "out");
    TORCH_CHECK(out->numel() == rows * width, "embed_scaled: out");
  }
  by_dtype(table, [&](auto tag) {
    using T = ELEM(tag);
    T* o = !out.has_value() || out->data_ptr() == residual.data_ptr()
        ? nullptr : ptr<T>(*out);
    launch_embed_scaled<T>(o, ptr<float>(residual), ptr<T>(table),
                           ids.data_ptr<long>(), (float)scale, rows,
                           (int)width, table.size(0), stream());
  });
}

void rms_scale(Tensor out, Tensor x, Tensor w, double eps) {
  const long width = w.numel(), rows = x.numel() / width;
  check_param(w, width, "norm weight");
  check_param(x, rows * width, "x");
  check(out, out.scalar_type(), "out");
  TORCH_CHECK(out.numel() == x.numel() && x.size(-1) == width,
              "rms_scale: shape");
  by_dtype(out, [&](auto tag) {
    using T = ELEM(tag);
    launch_rms_scale<T>(ptr<T>(out), ptr<float>(x), ptr<float>(w), rows,
                        (int)width, (float)eps, stream());
  });
}

void add_rms(Tensor out, Tensor residual, Tensor h, Tensor w, double eps) {
  const long width = w.numel(), rows = h.numel() / width;
  check_param(w, width, "norm weight");
  check_param(residual, rows * width, "residual");
  check(h, h.scalar_type(), "h");
  check(out, h.scalar_type(), "out");
  TORCH_CHECK(out.numel() == h.numel() && h.size(-1) == width,
              "add_rms: shape");
  by_dtype(h, [&](auto tag) {
    using T = ELEM(tag);
    T* o = out.data_ptr() == residual.data_ptr() ? nullptr : ptr<T>(out);
    launch_add_rms<T>(o, ptr<float>(residual), ptr<T>(h), ptr<float>(w), rows,
                      (int)width, (float)eps, stream());
  });
}

void rms_gate(Tensor y, Tensor o, Tensor g, Tensor w, Maybe ss, long total,
              double eps) {
  const long rows = o.size(0), n = o.size(1);
  check_param(o, rows * n, "o");
  check_param(w, n, "norm weight");
  check(y, g.scalar_type(), "y");
  TORCH_CHECK(y.numel() == rows * n && total >= n, "rms_gate: shape");
  check_rows(g, g.scalar_type(), rows, n, g.stride(0), "g");
  TORCH_CHECK(ss.has_value() || total == n, "rms_gate: sum of squares");
  if (ss.has_value()) check_param(*ss, rows, "sum of squares");
  by_dtype(g, [&](auto tag) {
    using T = ELEM(tag);
    launch_rms_gate<T>(ptr<T>(y), ptr<float>(o), ptr<T>(g), ptr<float>(w),
                       opt(ss), rows, (int)n, total, g.stride(0), (float)eps,
                       stream());
  });
}

void row_squares(Tensor ss, Tensor x) {
  check_param(x, x.numel(), "x");
  check_param(ss, x.size(0), "ss");
  launch_row_squares(ptr<float>(ss), ptr<float>(x), x.size(0),
                     (int)x.size(1), stream());
}

void gelu_gate(Tensor out, Tensor z, Tensor table, Tensor ids, long column) {
  const long rows = z.size(0), n = z.size(1);
  check(z, z.scalar_type(), "z");
  check(out, z.scalar_type(), "out");
  check(table, z.scalar_type(), "table");
  check(ids, torch::kInt64, "ids");
  TORCH_CHECK(out.numel() == rows * n && ids.numel() == rows &&
                  table.dim() == 2 && column >= 0 &&
                  column + n <= table.size(1), "gelu_gate: shape");
  by_dtype(z, [&](auto tag) {
    using T = ELEM(tag);
    launch_gelu_gate<T>(ptr<T>(out), ptr<T>(z), ptr<T>(table),
                        ids.data_ptr<long>(), rows, (int)n, table.size(1),
                        column, table.size(0), stream());
  });
}

// ---- latent attention -----------------------------------------------------

struct LatentDims {
  long H, D, E, rank, rot;
};

const float* sink_of(const Maybe& sink, long heads) {
  if (sink.has_value()) check_param(*sink, heads, "sink");
  return opt(sink);
}

// gate [rows, H], a column view
template <typename T>
const T* gate_of(const Maybe& gate, torch::ScalarType dt, long rows,
                 long heads) {
  if (!gate.has_value()) return nullptr;
  check_rows(*gate, dt, rows, heads, gate->stride(0), "gate");
  return ptr<T>(*gate);
}

long stride_of(const Maybe& t) { return t.has_value() ? t->stride(0) : 0; }

// q [T, H * (D + rot)], cache [NB, 16, rank + rot], uk [rank, H * D]
LatentDims latent_dims(const Tensor& q, const Tensor& cache, long rank,
                       long heads, long D, long E) {
  check(cache, q.scalar_type(), "cache");
  TORCH_CHECK(cache.dim() == 3 && cache.size(1) == 16 &&
                  cache.size(2) >= rank, "latent cache");
  const long rot = cache.size(2) - rank;
  check_rows(q, q.scalar_type(), q.size(0), heads * (D + rot), q.stride(0),
             "q");
  return {heads, D, E, rank, rot};
}

// out [T, H * E] as a column view: rows and base for 8-byte stores
bool out_fits(const Tensor& out) {
  return out.stride(0) % 4 == 0 &&
         reinterpret_cast<uintptr_t>(out.data_ptr()) % 8 == 0;
}

bool latent_fits(Tensor q, Tensor cache, Tensor uk, Tensor uv, Tensor out,
                 long heads) {
  const long rank = uk.size(0);
  return q.scalar_type() == torch::kBFloat16 && q.stride(0) % 8 == 0 &&
         aligned16(q) && out_fits(out) &&
         latent_sizes_fit((int)(uk.size(1) / heads), (int)(uv.size(0) / heads),
                          (int)rank, (int)(cache.size(2) - rank));
}

void latent_rope_append(Tensor q, Maybe kv, Maybe w, Tensor positions,
                        Tensor freqs, Tensor slot_mapping, Tensor cache,
                        long heads, long rank, double eps, double gain,
                        Maybe side_x, Maybe side_out) {
  const long rows = q.size(0), rot = 2 * freqs.numel();
  const auto dt = q.scalar_type();
  TORCH_CHECK(heads >= 1 && q.size(1) % heads == 0 &&
                  q.size(1) / heads >= rot, "latent_rope_append: heads");
  const long D = q.size(1) / heads - rot;
  check_rows(q, dt, rows, heads * (D + rot), q.stride(0), "q");
  check(positions, torch::kInt64, "positions");
  check(slot_mapping, torch::kInt64, "slot_mapping");
  check(freqs, torch::kFloat64, "freqs");
  TORCH_CHECK(positions.numel() == rows && slot_mapping.numel() == rows &&
                  rot <= 4096, "latent_rope_append: rows");
  if (kv.has_value()) {
    TORCH_CHECK(w.has_value(), "latent_rope_append: norm weight");
    check_param(*w, rank, "norm weight");
    check_rows(*kv, dt, rows, rank + rot, kv->stride(0), "kv");
    check(cache, dt, "cache");
    TORCH_CHECK(cache.size(-1) == rank + rot, "latent cache");
  }
  by_dtype(q, [&](auto tag) {
    using T = ELEM(tag);
    launch_latent_rope_append<T>(
        ptr<T>(q), kv.has_value() ? ptr<T>(*kv) : nullptr, opt(w),
        positions.data_ptr<long>(), freqs.data_ptr<double>(),
        slot_mapping.data_ptr<long>(), ptr<T>(cache), rows, (int)heads,
        (int)D, (int)rank, (int)rot, q.stride(0), stride_of(kv), (float)eps,
        (float)gain, side_of<T>(side_x, side_out, rows, dt), stream());
  });
}

void latent_gather(Tensor out, Tensor cache, Tensor slots) {
  check(out, torch::kBFloat16, "out");
  check(cache, torch::kBFloat16, "cache");
  check(slots, torch::kInt64, "slots");
  const long width = cache.size(-1);
  TORCH_CHECK(width % 8 == 0 && out.numel() == slots.numel() * width,
              "latent_gather: shape");
  launch_latent_gather(ptr<bf16>(out), ptr<bf16>(cache),
                       slots.data_ptr<long>(), slots.numel(), (int)width,
                       stream());
}

// qa[r, h] = W_uk[h]^T q[rows[r], h, :D];  qa [R, H, rank]
void latent_absorb(Tensor qa, Tensor q, Tensor uk, Maybe rows, long heads) {
  const auto dt = q.scalar_type();
  const long R = qa.size(0), rank = uk.size(0), D = uk.size(1) / heads;
  check(qa, dt, "qa");
  check(uk, dt, "uk");
  TORCH_CHECK(qa.dim() == 3 && qa.size(1) == heads && qa.size(2) == rank &&
                  uk.size(1) == heads * D && q.size(1) % heads == 0,
              "latent_absorb: shape");
  const long head = q.size(1) / heads;
  TORCH_CHECK(head >= D, "latent_absorb: q");
  check_rows(q, dt, q.size(0), heads * head, q.stride(0), "q");
  if (rows.has_value())
    check_ints(*rows, R, "rows");
  else
    TORCH_CHECK(R == q.size(0), "latent_absorb: rows");
  const bool fast = D % 8 == 0 && rank % 8 == 0 && head % 8 == 0 &&
                    q.stride(0) % 8 == 0 && aligned16(q) && aligned16(uk);
  by_dtype(q, [&](auto tag) {
    using T = ELEM(tag);
    launch_head_gemm<T>(ptr<T>(qa), ptr<T>(q), ptr<T>(uk), opt_int(rows),
                        nullptr, R, (int)heads, (int)rank, (int)D,
                        q.stride(0), head, heads * D, D, heads * rank, rank,
                        nullptr, 0, fast, stream());
  });
}

// out[rows[r], h] = W_uv[h] o[r, h] sigmoid(gate[rows[r], h]);
// o [R, H, rank], uv [H * E, rank]
void latent_values(Tensor out, Tensor o, Tensor uv, Maybe rows, Maybe gate) {
  const auto dt = o.scalar_type();
  const long R = o.size(0), H = o.size(1), rank = o.size(2);
  check_rows(out, dt, out.size(0), uv.size(0), out.stride(0), "out");
  check(o, dt, "o");
  check(uv, dt, "uv");
  TORCH_CHECK(uv.size(0) % H == 0 && uv.size(1) == rank &&
                  out.size(1) == uv.size(0), "latent_values: shape");
  const long E = uv.size(0) / H;
  if (rows.has_value())
    check_ints(*rows, R, "rows");
  else
    TORCH_CHECK(R == out.size(0), "latent_values: rows");
  by_dtype(o, [&](auto tag) {
    using T = ELEM(tag);
    launch_head_gemm<T>(ptr<T>(out), ptr<T>(o), ptr<T>(uv), nullptr,
                        opt_int(rows), R, (int)H, (int)E, (int)rank, H * rank,
                        rank, rank, E * rank, out.stride(0), E,
                        gate_of<T>(gate, dt, out.size(0), H), stride_of(gate),
                        E % 8 == 0 && rank % 8 == 0 && out_fits(out),
                        stream());
  });
}

LatentDims check_absorbed(const Tensor& o, const Tensor& qa, const Tensor& q,
                          const Tensor& cache, const Tensor& block_tables,
                          const Tensor& positions, const Maybe& rows,
                          const Maybe& row_seq, long window) {
  const auto dt = q.scalar_type();
  const long R = qa.size(0), H = qa.size(1), rank = qa.size(2);
  check(qa, dt, "qa");
  check(o, dt, "o");
  TORCH_CHECK(qa.dim() == 3 && o.numel() == qa.numel(), "latent_attn: o");
  const long rot = cache.size(2) - rank;
  const auto d = latent_dims(q, cache, rank, H, q.size(1) / H - rot, 0);
  check(block_tables, torch::kInt32, "block_tables");
  check(positions, torch::kInt64, "positions");
  TORCH_CHECK(positions.numel() == q.size(0) && window >= 1,
              "latent_attn: rows");
  if (rows.has_value())
    check_ints(*rows, R, "rows");
  else
    TORCH_CHECK(R == q.size(0), "latent_attn: rows");
  if (row_seq.has_value())
    check_ints(*row_seq, q.size(0), "row_seq");
  else
    TORCH_CHECK(block_tables.size(0) >= q.size(0), "latent_attn: tables");
  return d;
}

void latent_attn_general(Tensor o, Tensor qa, Tensor q, Tensor cache,
                         Tensor block_tables, Tensor positions, Maybe rows,
                         Maybe row_seq, long window, double scale,
                         Maybe sink) {
  const auto d = check_absorbed(o, qa, q, cache, block_tables, positions,
                                rows, row_seq, window);
  by_dtype(q, [&](auto tag) {
    using T = ELEM(tag);
    launch_latent_attn_general<T>(
        ptr<T>(o), ptr<T>(qa), ptr<T>(q), ptr<T>(cache),
        block_tables.data_ptr<int>(), positions.data_ptr<long>(),
        opt_int(rows), opt_int(row_seq), sink_of(sink, d.H), qa.size(0),
        (int)block_tables.size(1), (int)d.H, (int)d.D, (int)d.rank,
        (int)d.rot, (int)window, (float)scale, q.stride(0), stream());
  });
}

// split 1: o [R, H, rank] bf16; otherwise o is the partial results of
// latent_merge_values, [R, H, split, rank + 4] float
void latent_attn_decode(Tensor o, Tensor qa, Tensor q, Tensor cache,
                        Tensor block_tables, Tensor positions, Maybe rows,
                        Maybe row_seq, long split, long window, double scale,
                        Maybe sink) {
  const auto d = check_absorbed(split > 1 ? qa : o, qa, q, cache,
                                block_tables, positions, rows, row_seq,
                                window);
  TORCH_CHECK(q.scalar_type() == torch::kBFloat16 && q.stride(0) % 8 == 0 &&
                  aligned16(q) &&
                  latent_sizes_fit((int)d.D, 8, (int)d.rank, (int)d.rot),
              "latent_attn_decode: sizes");
  TORCH_CHECK(split >= 1 && split <= 16, "latent_attn_decode: split");
  if (split > 1)
    check_param(o, qa.size(0) * d.H * split * (d.rank + 4), "partial");
  launch_latent_attn_decode(
      split > 1 ? nullptr : ptr<bf16>(o), split > 1 ? ptr<float>(o) : nullptr,
      ptr<bf16>(qa), ptr<bf16>(q), ptr<bf16>(cache),
      block_tables.data_ptr<int>(), positions.data_ptr<long>(),
      opt_int(rows), opt_int(row_seq), sink_of(sink, d.H), qa.size(0),
      (int)block_tables.size(1), (int)d.H, (int)d.D, (int)d.rank, (int)d.rot,
      (int)window, (float)scale, q.stride(0), (int)split, stream());
}

// out[rows[r], h] = W_uv[h] (combined partial results of r and h)
//                   sigmoid(gate[rows[r], h])
void latent_merge_values(Tensor out, Tensor partial, Tensor uv, Maybe rows,
                         long R, long heads, long split, Maybe gate) {
  const auto dt = torch::kBFloat16;
  check_rows(out, dt, out.size(0), uv.size(0), out.stride(0), "out");
  check(uv, dt, "uv");
  const long E = uv.size(0) / heads, rank = uv.size(1);
  TORCH_CHECK(uv.size(0) == heads * E && out_fits(out) &&
                  latent_sizes_fit(8, (int)E, (int)rank, 8) && split >= 1 &&
                  split <= 16, "latent_merge_values: sizes");
  check_param(partial, R * heads * split * (rank + 4), "partial");
  if (rows.has_value())
    check_ints(*rows, R, "rows");
  else
    TORCH_CHECK(R == out.size(0), "latent_merge_values: rows");
  launch_latent_merge_values(ptr<bf16>(out), ptr<float>(partial),
                             ptr<bf16>(uv), opt_int(rows), R, (int)split,
                             (int)heads, (int)E, (int)rank, out.stride(0),
                             gate_of<bf16>(gate, dt, out.size(0), heads),
                             stride_of(gate), stream());
}

void latent_attn_prefill(Tensor out, Tensor q, Tensor kn, Tensor lat,
                         Tensor vt, Tensor positions, Tensor seq_start,
                         Tensor kv_start, Tensor kv_first, Tensor tiles,
                         long heads, long window, double scale, Maybe sink,
                         Maybe gate) {
  const auto dt = torch::kBFloat16;
  check(kn, dt, "kn");
  check(lat, dt, "lat");
  check(vt, dt, "vt");
  const long nkv = lat.size(0), D = kn.size(1) / heads;
  const long E = vt.size(0) / heads;
  TORCH_CHECK(kn.size(0) == nkv && vt.size(1) == nkv && nkv % 8 == 0 &&
                  kn.size(1) == heads * D && vt.size(0) == heads * E &&
                  q.size(1) % heads == 0, "latent_attn_prefill: keys");
  const long rot = q.size(1) / heads - D, rank = lat.size(1) - rot;
  TORCH_CHECK(rot >= 0 && rank >= 1 && q.stride(0) % 8 == 0 && aligned16(q) &&
                  latent_sizes_fit((int)D, (int)E, (int)rank, (int)rot),
              "latent_attn_prefill: sizes");
  check_rows(q, dt, q.size(0), heads * (D + rot), q.stride(0), "q");
  check_rows(out, dt, q.size(0), heads * E, out.stride(0), "out");
  TORCH_CHECK(out_fits(out) && window >= 1, "latent_attn_prefill: out");
  check(positions, torch::kInt64, "positions");
  TORCH_CHECK(positions.numel() == q.size(0), "latent_attn_prefill: rows");
  const long B = seq_start.numel() - 1;
  check_tiles(tiles, seq_start, B);
  TORCH_CHECK(tiles.size(0) <= 65535, "latent_attn_prefill: tiles");
  check_ints(kv_start, B, "kv_start");
  check_ints(kv_first, B, "kv_first");
  launch_latent_attn_prefill(
      ptr<bf16>(out), ptr<bf16>(q), ptr<bf16>(kn), ptr<bf16>(lat),
      ptr<bf16>(vt), positions.data_ptr<long>(), seq_start.data_ptr<int>(),
      kv_start.data_ptr<int>(), kv_first.data_ptr<int>(),
      tiles.data_ptr<int>(), sink_of(sink, heads), (int)tiles.size(0),
      (int)heads, (int)D, (int)E, (int)rank, (int)rot, nkv, (int)window,
      (float)scale, q.stride(0), out.stride(0),
      gate_of<bf16>(gate, dt, q.size(0), heads), stride_of(gate), stream());
}

// ---- experts --------------------------------------------------------------

// logits [T, N] or, with a shared expert, [T, N + 1], N = E + identity; true:
// shared
bool check_route(const Tensor& weight, const Tensor& logits, long E, long top,
                 const Maybe& correction, long identity) {
  check(logits, torch::kFloat32, "logits");
  TORCH_CHECK(logits.dim() == 2, "experts: logits");
  const long N = E + identity;
  const long T = logits.size(0), extra = logits.size(1) - N;
  TORCH_CHECK(extra == 0 || extra == 1, "experts: logits");
  TORCH_CHECK(E >= 1 && identity >= 0 && N <= 1024 && top >= 1 && top <= 63 &&
                  top <= N,
              "experts: at most 1024 experts, of which at most 63 at once");
  if (correction.has_value()) check_param(*correction, N, "correction");
  check_param(weight, T * (top + extra), "weight");
  return extra == 1;
}

void experts_route(Tensor weight, Tensor ids, Tensor logits, long E, long top,
                   Maybe correction, long identity) {
  const bool shared = check_route(weight, logits, E, top, correction,
                                  identity);
  check_ints(ids, logits.size(0) * top, "ids");
  launch_experts_route(ptr<float>(weight), ids.data_ptr<int>(),
                       ptr<float>(logits), (int)logits.size(0), (int)E,
                       (int)top, shared, false, (int)identity,
                       opt(correction), stream());
}

void check_sorted(const Tensor& order, const Tensor& expert,
                  const Tensor& place, long choices, long kinds, long bm) {
  const long tiles = expert.numel();
  check_ints(order, tiles * bm, "order");
  check_ints(expert, tiles, "expert");
  check_ints(place, choices, "place");
  // enough tiles however the choices fall
  TORCH_CHECK(tiles >= std::min(choices, (choices + kinds * (bm - 1)) / bm),
              "experts: tiles");
}

void experts_sort(Tensor order, Tensor expert, Tensor place, Tensor ids,
                  long kinds, long bm) {
  check_ints(ids, ids.numel(), "ids");
  check_sorted(order, expert, place, ids.numel(), kinds, bm);
  TORCH_CHECK(kinds >= 1 && kinds <= 1025, "experts_sort: kinds");
  launch_experts_sort(order.data_ptr<int>(), expert.data_ptr<int>(),
                      place.data_ptr<int>(), ids.data_ptr<int>(),
                      (int)ids.numel(), (int)kinds, (int)bm,
                      (int)expert.numel(), stream());
}

void experts_route_sort(Tensor weight, Tensor ids, Tensor place, Tensor order,
                        Tensor expert, Tensor logits, long bm, long E,
                        long top, Maybe correction, long identity) {
  const bool shared = check_route(weight, logits, E, top, correction,
                                  identity);
  const long T = logits.size(0), choices = T * (top + shared);
  check_ints(ids, choices, "ids");
  check_sorted(order, expert, place, choices, E + shared, bm);
  launch_experts_route_sort(
      ptr<float>(weight), ids.data_ptr<int>(), place.data_ptr<int>(),
      order.data_ptr<int>(), expert.data_ptr<int>(), ptr<float>(logits),
      (int)T, (int)E, (int)top, shared, (int)bm, (int)expert.numel(),
      (int)identity, opt(correction), stream());
}

void experts_gemm(bool up, const Tensor& out, const Tensor& x,
                  const Tensor& w, const Maybe& ws, const Tensor& order,
                  const Tensor& expert, long div, c10::optional<double> limit,
                  long bm) {
  const auto dt = x.scalar_type();
  check(out, dt, "out");
  check(x, dt, "x");
  check(w, dt, "w");
  TORCH_CHECK(w.dim() == 3 && x.dim() == 2 && out.dim() == 2,
              "experts: shape");
  const long E = w.size(0), N = up ? w.size(1) / 2 : w.size(1);
  const long K = w.size(2);
  long Ns = 0, Ks = 0;
  if (ws.has_value()) {
    check(*ws, dt, "shared weight");
    TORCH_CHECK(ws->dim() == 3 && ws->size(0) == 1, "experts: shared");
    Ns = up ? ws->size(1) / 2 : ws->size(1);
    Ks = ws->size(2);
    TORCH_CHECK(up ? Ks == K : Ns == N, "experts: shared");
  }
  const long tiles = expert.numel();
  check_ints(order, tiles * bm, "order");
  check_ints(expert, tiles, "expert");
  TORCH_CHECK(out.size(0) == tiles * bm && out.size(1) >= std::max(N, Ns) &&
                  x.size(1) >= std::max(K, Ks) &&
                  (up ? div >= 1 : x.size(0) == tiles * bm),
              "experts: rows");
  TORCH_CHECK(bm == 1 || bm == 16 || bm == 32 || bm == 64, "experts: bm");
  if (bm != 1)
    TORCH_CHECK(dt == torch::kBFloat16 && N % 8 == 0 && K % 8 == 0 &&
                    Ns % 8 == 0 && Ks % 8 == 0 && x.size(1) % 8 == 0 &&
                    out.size(1) % 8 == 0 && tiles <= 65535,
                "experts: sizes");
  by_dtype(x, [&](auto tag) {
    using T = ELEM(tag);
    launch_experts_gemm<T>(up, ptr<T>(out), ptr<T>(x), ptr<T>(w),
                           ws.has_value() ? ptr<T>(*ws) : nullptr,
                           order.data_ptr<int>(), expert.data_ptr<int>(),
                           (int)tiles, (int)E, (int)N, (int)K, (int)Ns,
                           (int)Ks, (int)div, x.size(1), out.size(1), (int)bm,
                           limit.has_value(), (float)limit.value_or(0.),
                           stream());
  });
}

void experts_up(Tensor h, Tensor x, Tensor w, Maybe ws, Tensor order,
                Tensor expert, long div, c10::optional<double> limit,
                long bm) {
  experts_gemm(true, h, x, w, ws, order, expert, div, limit, bm);
}

void experts_down(Tensor y, Tensor h, Tensor w, Maybe ws, Tensor order,
                  Tensor expert, long bm) {
  experts_gemm(false, y, h, w, ws, order, expert, 1, c10::nullopt, bm);
}

void experts_sum(Tensor out, Tensor y, Tensor place, Tensor weight,
                 Maybe shared, Maybe identity, Maybe residual, Maybe w,
                 double eps) {
  const auto dt = y.scalar_type();
  check(y, dt, "y");
  check(out, dt, "out");
  check(place, torch::kInt32, "place");
  TORCH_CHECK(place.dim() == 2 && out.dim() == 2, "experts_sum: shape");
  const long rows = place.size(0), n = place.size(1), width = y.size(1);
  TORCH_CHECK(out.size(0) == rows && out.size(1) == width,
              "experts_sum: out");
  check_param(weight, rows * (n + (shared.has_value() ? 1 : 0)), "weight");
  if (shared.has_value()) {
    check(*shared, dt, "shared");
    TORCH_CHECK(shared->numel() == rows * width, "experts_sum: shared");
  }
  if (identity.has_value()) {
    check(*identity, dt, "identity");
    TORCH_CHECK(identity->numel() == rows * width, "experts_sum: identity");
  }
  if (residual.has_value()) {
    check_param(*residual, rows * width, "residual");
    TORCH_CHECK(w.has_value(), "experts_sum: norm weight");
    check_param(*w, width, "norm weight");
  }
  by_dtype(y, [&](auto tag) {
    using T = ELEM(tag);
    T* o = residual.has_value() && out.data_ptr() == residual->data_ptr()
        ? nullptr : ptr<T>(out);
    launch_experts_sum<T>(
        o, opt(residual), ptr<T>(y),
        shared.has_value() ? ptr<T>(*shared) : nullptr,
        identity.has_value() ? ptr<T>(*identity) : nullptr,
        ptr<float>(weight), place.data_ptr<int>(), opt(w), rows, (int)n,
        (int)width, (float)eps, stream());
  });
}

}  // namespace

void register_latent(pybind11::module_& m) {
  m.def("embed_scaled", &embed_scaled);
  m.def("rms_scale", &rms_scale);
  m.def("add_rms", &add_rms);
  m.def("rms_gate", &rms_gate);
  m.def("row_squares", &row_squares);
  m.def("gelu_gate", &gelu_gate);
  m.def("latent_fits", &latent_fits);
  m.def("latent_rope_append", &latent_rope_append);
  m.def("latent_gather", &latent_gather);
  m.def("latent_absorb", &latent_absorb);
  m.def("latent_values", &latent_values);
  m.def("latent_attn_general", &latent_attn_general);
  m.def("latent_attn_decode", &latent_attn_decode);
  m.def("latent_merge_values", &latent_merge_values);
  m.def("latent_attn_prefill", &latent_attn_prefill);
  namespace py = pybind11;
  m.def("experts_route", &experts_route, py::arg("weight"), py::arg("ids"),
        py::arg("logits"), py::arg("E"), py::arg("top"),
        py::arg("correction") = py::none(), py::arg("identity") = 0);
  m.def("experts_sort", &experts_sort);
  m.def("experts_route_sort", &experts_route_sort);
  m.def("experts_up", &experts_up);
  m.def("experts_down", &experts_down);
  m.def("experts_sum", &experts_sum);
}
