// Bindings of sublayer inputs, head norms, chunked sigmoid attention and
// windowed attention with kept tokens (conv.hip, kv_norm.hip, rope_norm.hip,
// attn_sigmoid.hip, attn_kept.hip, the activations of act.hip and the closing
// step of experts.hip).
#include "bindings.h"
#include "sublayer.h"

template <typename T>
void launch_add_rms_next(const Between<T>&, const T*, long, hipStream_t);
template <typename T>
void launch_causal_conv(T*, const T*, const float*, T*, const int*,
                        const long*, const int*, const int*, int, int, int,
                        int, hipStream_t);
template <typename T>
void launch_experts_sum_next(const Between<T>&, const T*, const T*, const T*,
                             const float*, const int*, long, int,
                             hipStream_t);
template <typename T>
void launch_norm_append(T*, const T*, const T*, const float*, const float*,
                        const long*, T*, T*, long, int, int, int, int, int,
                        long, long, long, float, hipStream_t);
template <typename T>
void launch_sigmoid_attn_general(T*, const T*, const T*, const T*, const int*,
                                 const long*, const int*, const float*, long,
                                 int, int, int, int, int, int, float, float,
                                 long, hipStream_t);
void launch_sigmoid_attn_prefill(bf16*, const bf16*, const bf16*, const bf16*,
                                 const int*, const long*, const int*,
                                 const int*, const float*, int, int, int, int,
                                 int, int, int, float, float, long,
                                 hipStream_t);
void launch_sigmoid_attn_decode(bf16*, const bf16*, const bf16*, const bf16*,
                                const int*, const long*, const float*, float*,
                                long, int, int, int, int, int, int, float,
                                float, long, int, hipStream_t);
template <typename T>
void launch_rope_norm_append(T*, const T*, const T*, const long*,
                             const double*, const double*, const long*, T*,
                             T*, long, int, int, int, int, int, int, int,
                             long, long, long, float, float, bool,
                             const SideRelu<T>&, hipStream_t);
template <typename T>
void launch_kept_attn_general(T*, const T*, const T*, const T*, const int*,
                              const long*, const int*, const double*,
                              const float*, long, int, int, int, int, int,
                              int, int, float, long, long, hipStream_t);
void launch_kept_attn_prefill(bf16*, const bf16*, const bf16*, const bf16*,
                              const int*, const long*, const int*, const int*,
                              const double*, const float*, int, int, int, int,
                              int, int, int, int, float, bool, long, long,
                              hipStream_t);
void launch_kept_attn_decode(bf16*, const bf16*, const bf16*, const bf16*,
                             const int*, const long*, const double*,
                             const float*, float*, long, int, int, int, int,
                             int, int, int, float, bool, long, long, int,
                             hipStream_t);
template <typename T>
void launch_clamped_glu(T*, const T*, long, int, float, hipStream_t);
template <typename T> void launch_squared_relu(T*, long, hipStream_t);

namespace {

using torch::Tensor;
using Maybe = c10::optional<Tensor>;

// ---- between sublayers ----------------------------------------------------

// tail [slots, taps - 1, width] of conv [taps, width]
void check_conv(const Tensor& conv, const Tensor& tail, const Tensor& slots,
                long width, torch::ScalarType dt) {
  TORCH_CHECK(conv.dim() == 2 && conv.size(0) >= 1, "conv");
  check_param(conv, conv.size(0) * width, "conv");
  check(tail, dt, "tail");
  check(slots, torch::kInt32, "slots");
  TORCH_CHECK(tail.dim() == 3 && tail.size(1) == conv.size(0) - 1 &&
                  tail.size(2) == width, "conv tail");
}

template <typename T>
Between<T> between(const Tensor& out, const Tensor& residual, const Maybe& w,
                   const Tensor& pre, double eps, const Maybe& conv,
                   const Maybe& tail, const Maybe& slots,
                   const Maybe& positions) {
  const long width = pre.numel(), rows = residual.numel() / width;
  const auto dt = out.scalar_type();
  check(out, dt, "out");
  check_param(pre, width, "norm weight");
  check_param(residual, rows * width, "residual");
  if (w.has_value()) check_param(*w, width, "norm weight");
  TORCH_CHECK(out.numel() == rows * width && residual.size(-1) == width,
              "add_rms_next: shape");
  Between<T> a{ptr<T>(out), ptr<float>(residual), opt(w), ptr<float>(pre),
               nullptr, nullptr, nullptr, nullptr, 0, (int)width, (float)eps};
  if (conv.has_value()) {
    TORCH_CHECK(tail.has_value() && slots.has_value() &&
                    positions.has_value(), "add_rms_next: conv");
    check_conv(*conv, *tail, *slots, width, dt);
    check(*positions, torch::kInt64, "positions");
    TORCH_CHECK(slots->numel() == rows && positions->numel() == rows,
                "add_rms_next: rows");
    a.conv = ptr<float>(*conv);
    a.tail = ptr<T>(*tail);
    a.slots = slots->data_ptr<int>();
    a.positions = positions->data_ptr<long>();
    a.taps = (int)conv->size(0);
  }
  return a;
}

void add_rms_next(Tensor out, Tensor residual, Maybe y, Maybe w, Tensor pre,
                  double eps, Maybe conv, Maybe tail, Maybe slots,
                  Maybe positions) {
  TORCH_CHECK(y.has_value() || !w.has_value(), "add_rms_next: y");
  if (y.has_value()) {
    check(*y, out.scalar_type(), "y");
    TORCH_CHECK(y->numel() == residual.numel(), "add_rms_next: y");
  }
  by_dtype(out, [&](auto tag) {
    using T = ELEM(tag);
    const auto a = between<T>(out, residual, w, pre, eps, conv, tail, slots,
                              positions);
    launch_add_rms_next<T>(a, y.has_value() ? ptr<T>(*y) : nullptr,
                           residual.numel() / pre.numel(), stream());
  });
}

void experts_sum_next(Tensor out, Tensor y, Tensor place, Tensor weight,
                      Maybe shared, Maybe identity, Tensor residual, Tensor w,
                      Tensor pre, double eps, Maybe conv, Maybe tail,
                      Maybe slots, Maybe positions) {
  const auto dt = out.scalar_type();
  check(y, dt, "y");
  check(place, torch::kInt32, "place");
  TORCH_CHECK(place.dim() == 2 && y.size(-1) == pre.numel(),
              "experts_sum_next: shape");
  const long rows = place.size(0), n = place.size(1);
  TORCH_CHECK(residual.numel() == rows * pre.numel(),
              "experts_sum_next: rows");
  check_param(weight, rows * (n + (shared.has_value() ? 1 : 0)), "weight");
  for (const Maybe& t : {shared, identity})
    if (t.has_value()) {
      check(*t, dt, "expert rows");
      TORCH_CHECK(t->numel() == residual.numel(), "experts_sum_next: rows");
    }
  by_dtype(out, [&](auto tag) {
    using T = ELEM(tag);
    const auto a = between<T>(out, residual, w, pre, eps, conv, tail, slots,
                              positions);
    launch_experts_sum_next<T>(
        a, ptr<T>(y), shared.has_value() ? ptr<T>(*shared) : nullptr,
        identity.has_value() ? ptr<T>(*identity) : nullptr,
        ptr<float>(weight), place.data_ptr<int>(), rows, (int)n, stream());
  });
}

void causal_conv(Tensor out, Tensor h, Tensor w, Tensor tail,
                 Tensor seq_start, Tensor positions, Tensor slots,
                 Tensor tiles) {
  const auto dt = h.scalar_type();
  check(h, dt, "h");
  check(out, dt, "out");
  TORCH_CHECK(h.dim() == 2 && out.numel() == h.numel() &&
                  out.data_ptr() != h.data_ptr(), "causal_conv: shape");
  check_conv(w, tail, slots, h.size(1), dt);
  check_tiles(tiles, seq_start, slots.numel());
  check(positions, torch::kInt64, "positions");
  TORCH_CHECK(positions.numel() == h.size(0), "causal_conv: rows");
  by_dtype(h, [&](auto tag) {
    using T = ELEM(tag);
    launch_causal_conv<T>(
        ptr<T>(out), ptr<T>(h), ptr<float>(w), ptr<T>(tail),
        seq_start.data_ptr<int>(), positions.data_ptr<long>(),
        slots.data_ptr<int>(), tiles.data_ptr<int>(), (int)tiles.size(0),
        (int)slots.numel(), (int)w.size(0), (int)h.size(1), stream());
  });
}

// ---- activations ----------------------------------------------------------

void clamped_glu(Tensor out, Tensor x, double limit) {
  check(x, x.scalar_type(), "x");
  check(out, x.scalar_type(), "out");
  const long inter = out.size(-1), rows = inter ? out.numel() / inter : 0;
  TORCH_CHECK(x.size(-1) == 2 * inter && x.numel() == 2 * out.numel(),
              "clamped_glu: shape");
  by_dtype(x, [&](auto tag) {
    using T = ELEM(tag);
    launch_clamped_glu<T>(ptr<T>(out), ptr<T>(x), rows, (int)inter,
                          (float)limit, stream());
  });
}

void squared_relu(Tensor x) {
  check(x, x.scalar_type(), "x");
  by_dtype(x, [&](auto tag) {
    using T = ELEM(tag);
    launch_squared_relu<T>(ptr<T>(x), x.numel(), stream());
  });
}

// ---- attention ------------------------------------------------------------

struct HeadDims { int H, G, D, E; };

// q [T, H * D] rows, k_cache [NB, G, 16, D], v_cache [NB, G, E, 16]
HeadDims check_heads(const Tensor& q, const Tensor& k_cache,
                     const Tensor& v_cache) {
  const auto dt = q.scalar_type();
  check(k_cache, dt, "k_cache");
  check(v_cache, dt, "v_cache");
  TORCH_CHECK(k_cache.dim() == 4 && v_cache.dim() == 4 &&
                  k_cache.size(0) == v_cache.size(0) &&
                  k_cache.size(1) == v_cache.size(1) &&
                  k_cache.size(2) == 16 && v_cache.size(3) == 16,
              "cache: k [NB, G, 16, D], v [NB, G, E, 16]");
  const long G = k_cache.size(1), D = k_cache.size(3);
  TORCH_CHECK(q.dim() == 2 && q.size(1) % (D * G) == 0, "q: head groups");
  check_rows(q, dt, q.size(0), q.size(1), q.stride(0), "q");
  return {(int)(q.size(1) / D), (int)G, (int)D, (int)v_cache.size(2)};
}

void norm_append(Tensor q, Tensor k, Tensor v, Tensor qw, Tensor kw,
                 Tensor slot_mapping, Tensor k_cache, Tensor v_cache,
                 double eps) {
  const auto dt = q.scalar_type();
  const auto d = check_heads(q, k_cache, v_cache);
  const long rows = q.size(0);
  check_rows(k, dt, rows, (long)d.G * d.D, k.stride(0), "k");
  check_rows(v, dt, rows, (long)d.G * d.E, v.stride(0), "v");
  check_param(qw, d.D, "query norm");
  check_param(kw, d.D, "key norm");
  check(slot_mapping, torch::kInt64, "slot_mapping");
  TORCH_CHECK(slot_mapping.numel() == rows, "norm_append: rows");
  by_dtype(q, [&](auto tag) {
    using T = ELEM(tag);
    launch_norm_append<T>(
        ptr<T>(q), ptr<T>(k), ptr<T>(v), ptr<float>(qw), ptr<float>(kw),
        slot_mapping.data_ptr<long>(), ptr<T>(k_cache), ptr<T>(v_cache), rows,
        d.H, d.G, d.D, d.E, 16, q.stride(0), k.stride(0), v.stride(0),
        (float)eps, stream());
  });
}

// 16-byte loads of q (rows and base), sizes of the padded kernels
bool sigmoid_attn_fits(Tensor q, Tensor k_cache, Tensor v_cache) {
  const long D = k_cache.size(3), E = v_cache.size(2);
  return q.scalar_type() == torch::kBFloat16 && D % 8 == 0 && E % 8 == 0 &&
         D <= 256 && E <= 256 && q.stride(0) % 8 == 0 &&
         reinterpret_cast<uintptr_t>(q.data_ptr()) % 16 == 0;
}

HeadDims check_attention(const Tensor& out, const Tensor& q,
                         const Tensor& k_cache, const Tensor& v_cache,
                         const Tensor& block_tables, const Tensor& positions,
                         const Tensor& bias, long chunk, double cap) {
  const auto d = check_heads(q, k_cache, v_cache);
  check(out, q.scalar_type(), "out");
  TORCH_CHECK(out.numel() == q.size(0) * d.H * d.E, "sigmoid_attn: out");
  check(block_tables, torch::kInt32, "block_tables");
  check(positions, torch::kInt64, "positions");
  TORCH_CHECK(positions.numel() == q.size(0) && chunk >= 1 &&
                  chunk <= INT_MAX && cap > 0, "sigmoid_attn: rows, chunk");
  check_param(bias, d.H, "bias");
  return d;
}

void sigmoid_attn_general(Tensor out, Tensor q, Tensor k_cache,
                          Tensor v_cache, Tensor block_tables,
                          Tensor positions, Maybe row_seq, Tensor bias,
                          long chunk, double scale, double cap) {
  const auto d = check_attention(out, q, k_cache, v_cache, block_tables,
                                 positions, bias, chunk, cap);
  const long rows = q.size(0);
  TORCH_CHECK(d.E <= 1024 && d.D <= 8192, "sigmoid_attn: head sizes");
  const int* rs = nullptr;
  if (row_seq.has_value()) {
    check(*row_seq, torch::kInt32, "row_seq");
    TORCH_CHECK(row_seq->numel() == rows, "sigmoid_attn: row_seq");
    rs = row_seq->data_ptr<int>();
  } else {
    TORCH_CHECK(block_tables.size(0) >= rows, "sigmoid_attn: block_tables");
  }
  by_dtype(q, [&](auto tag) {
    using T = ELEM(tag);
    launch_sigmoid_attn_general<T>(
        ptr<T>(out), ptr<T>(q), ptr<T>(k_cache), ptr<T>(v_cache),
        block_tables.data_ptr<int>(), positions.data_ptr<long>(), rs,
        ptr<float>(bias), rows, (int)block_tables.size(1), d.H, d.G, d.D, d.E,
        (int)chunk, (float)scale, (float)cap, q.stride(0), stream());
  });
}

void sigmoid_attn_prefill(Tensor out, Tensor q, Tensor k_cache,
                          Tensor v_cache, Tensor block_tables,
                          Tensor positions, Tensor seq_start, Tensor tiles,
                          Tensor bias, long chunk, double scale, double cap) {
  const auto d = check_attention(out, q, k_cache, v_cache, block_tables,
                                 positions, bias, chunk, cap);
  TORCH_CHECK(sigmoid_attn_fits(q, k_cache, v_cache), "sigmoid_attn: sizes");
  check_tiles(tiles, seq_start, block_tables.size(0));
  TORCH_CHECK(tiles.size(0) <= 65535, "sigmoid_attn: tiles");
  launch_sigmoid_attn_prefill(
      ptr<bf16>(out), ptr<bf16>(q), ptr<bf16>(k_cache), ptr<bf16>(v_cache),
      block_tables.data_ptr<int>(), positions.data_ptr<long>(),
      seq_start.data_ptr<int>(), tiles.data_ptr<int>(), ptr<float>(bias),
      (int)tiles.size(0), (int)block_tables.size(1), d.H, d.G, d.D, d.E,
      (int)chunk, (float)scale, (float)cap, q.stride(0), stream());
}

void sigmoid_attn_decode(Tensor out, Tensor q, Tensor k_cache, Tensor v_cache,
                         Tensor block_tables, Tensor positions, Tensor bias,
                         Maybe partial, long split, long chunk, double scale,
                         double cap) {
  const auto d = check_attention(out, q, k_cache, v_cache, block_tables,
                                 positions, bias, chunk, cap);
  const long rows = q.size(0);
  TORCH_CHECK(sigmoid_attn_fits(q, k_cache, v_cache), "sigmoid_attn: sizes");
  TORCH_CHECK(block_tables.size(0) >= rows && split >= 1 && split <= 64,
              "sigmoid_attn_decode: rows, split");
  if (split > 1) {
    TORCH_CHECK(partial.has_value(), "sigmoid_attn_decode: partial");
    check_param(*partial, rows * d.H * split * d.E, "partial");
  }
  launch_sigmoid_attn_decode(
      ptr<bf16>(out), ptr<bf16>(q), ptr<bf16>(k_cache), ptr<bf16>(v_cache),
      block_tables.data_ptr<int>(), positions.data_ptr<long>(),
      ptr<float>(bias), split > 1 ? ptr<float>(*partial) : nullptr, rows,
      (int)block_tables.size(1), d.H, d.G, d.D, d.E, (int)chunk, (float)scale,
      (float)cap, q.stride(0), (int)split, stream());
}

// freqs [rot / 2] and turn [E / 2 or none] float64
void rope_norm_append(Tensor q, Tensor k, Tensor v, Tensor positions,
                      Tensor freqs, Tensor turn, Tensor slot_mapping,
                      Tensor k_cache, Tensor v_cache, double gain,
                      c10::optional<double> eps, Maybe side_x,
                      Maybe side_out) {
  const auto dt = q.scalar_type();
  const auto d = check_heads(q, k_cache, v_cache);
  const long rows = q.size(0);
  check_rows(k, dt, rows, (long)d.G * d.D, k.stride(0), "k");
  check_rows(v, dt, rows, (long)d.G * d.E, v.stride(0), "v");
  check(positions, torch::kInt64, "positions");
  check(slot_mapping, torch::kInt64, "slot_mapping");
  check(freqs, torch::kFloat64, "freqs");
  check(turn, torch::kFloat64, "turn");
  const long rot = 2 * freqs.numel(), vrot = 2 * turn.numel();
  TORCH_CHECK(positions.numel() == rows && slot_mapping.numel() == rows,
              "rope_norm_append: rows");
  TORCH_CHECK(rot <= d.D && (vrot == 0 || vrot == d.E) && rot + vrot <= 8192,
              "rope_norm_append: rotated sizes");
  by_dtype(q, [&](auto tag) {
    using T = ELEM(tag);
    launch_rope_norm_append<T>(
        ptr<T>(q), ptr<T>(k), ptr<T>(v), positions.data_ptr<long>(),
        freqs.data_ptr<double>(), turn.data_ptr<double>(),
        slot_mapping.data_ptr<long>(), ptr<T>(k_cache), ptr<T>(v_cache), rows,
        d.H, d.G, d.D, d.E, (int)rot, (int)vrot, 16, q.stride(0), k.stride(0),
        v.stride(0), (float)gain, (float)eps.value_or(0.0), eps.has_value(),
        side_of<T>(side_x, side_out, rows, dt), stream());
  });
}

// 16-byte loads of q and 8-byte stores of out (rows and bases), sizes of the
// padded kernels
bool kept_attn_fits(Tensor out, Tensor q, Tensor k_cache, Tensor v_cache) {
  return sigmoid_attn_fits(q, k_cache, v_cache) && out.stride(0) % 4 == 0 &&
         reinterpret_cast<uintptr_t>(out.data_ptr()) % 8 == 0;
}

struct KeptArgs {
  HeadDims d;
  const double* turn;
  const float* sink;
};

KeptArgs check_kept(const Tensor& out, const Tensor& q, const Tensor& k_cache,
                    const Tensor& v_cache, const Tensor& block_tables,
                    const Tensor& positions, const Tensor& turn,
                    const Maybe& sink, long window, long keep) {
  const auto d = check_heads(q, k_cache, v_cache);
  check_rows(out, q.scalar_type(), q.size(0), (long)d.H * d.E, out.stride(0),
             "out");
  check(block_tables, torch::kInt32, "block_tables");
  check(positions, torch::kInt64, "positions");
  check(turn, torch::kFloat64, "turn");
  TORCH_CHECK(turn.numel() == 0 || 2 * turn.numel() == d.E,
              "kept_attn: turn");
  constexpr long most = 1L << 30;
  TORCH_CHECK(positions.numel() == q.size(0) && window >= 1 &&
                  window <= most && keep >= 0 && keep <= most,
              "kept_attn: rows, window");
  if (sink.has_value()) check_param(*sink, d.H, "sink");
  return {d, turn.numel() ? turn.data_ptr<double>() : nullptr, opt(sink)};
}

void kept_attn_general(Tensor out, Tensor q, Tensor k_cache, Tensor v_cache,
                       Tensor block_tables, Tensor positions, Maybe row_seq,
                       Tensor turn, Maybe sink, long window, long keep,
                       double scale) {
  const auto a = check_kept(out, q, k_cache, v_cache, block_tables, positions,
                            turn, sink, window, keep);
  const long rows = q.size(0);
  TORCH_CHECK(a.d.E <= 1024 && a.d.D <= 8192, "kept_attn: head sizes");
  const int* rs = nullptr;
  if (row_seq.has_value()) {
    check(*row_seq, torch::kInt32, "row_seq");
    TORCH_CHECK(row_seq->numel() == rows, "kept_attn: row_seq");
    rs = row_seq->data_ptr<int>();
  } else {
    TORCH_CHECK(block_tables.size(0) >= rows, "kept_attn: block_tables");
  }
  by_dtype(q, [&](auto tag) {
    using T = ELEM(tag);
    launch_kept_attn_general<T>(
        ptr<T>(out), ptr<T>(q), ptr<T>(k_cache), ptr<T>(v_cache),
        block_tables.data_ptr<int>(), positions.data_ptr<long>(), rs, a.turn,
        a.sink, rows, (int)block_tables.size(1), a.d.H, a.d.G, a.d.D, a.d.E,
        (int)window, (int)keep, (float)scale, q.stride(0), out.stride(0),
        stream());
  });
}

void kept_attn_prefill(Tensor out, Tensor q, Tensor k_cache, Tensor v_cache,
                       Tensor block_tables, Tensor positions,
                       Tensor seq_start, Tensor tiles, Tensor turn,
                       Maybe sink, long window, long keep, double scale,
                       bool bounded) {
  const auto a = check_kept(out, q, k_cache, v_cache, block_tables, positions,
                            turn, sink, window, keep);
  TORCH_CHECK(kept_attn_fits(out, q, k_cache, v_cache), "kept_attn: sizes");
  check_tiles(tiles, seq_start, block_tables.size(0));
  TORCH_CHECK(tiles.size(0) <= 65535, "kept_attn: tiles");
  launch_kept_attn_prefill(
      ptr<bf16>(out), ptr<bf16>(q), ptr<bf16>(k_cache), ptr<bf16>(v_cache),
      block_tables.data_ptr<int>(), positions.data_ptr<long>(),
      seq_start.data_ptr<int>(), tiles.data_ptr<int>(), a.turn, a.sink,
      (int)tiles.size(0), (int)block_tables.size(1), a.d.H, a.d.G, a.d.D,
      a.d.E, (int)window, (int)keep, (float)scale, bounded, q.stride(0),
      out.stride(0), stream());
}

// partial [rows, H, split, E + 4] float where split > 1
void kept_attn_decode(Tensor out, Tensor q, Tensor k_cache, Tensor v_cache,
                      Tensor block_tables, Tensor positions, Tensor turn,
                      Maybe sink, Maybe partial, long split, long window,
                      long keep, double scale, bool bounded) {
  const auto a = check_kept(out, q, k_cache, v_cache, block_tables, positions,
                            turn, sink, window, keep);
  const long rows = q.size(0);
  TORCH_CHECK(kept_attn_fits(out, q, k_cache, v_cache), "kept_attn: sizes");
  TORCH_CHECK(block_tables.size(0) >= rows && split >= 1 && split <= 64,
              "kept_attn_decode: rows, split");
  if (split > 1) {
    TORCH_CHECK(partial.has_value(), "kept_attn_decode: partial");
    check_param(*partial, rows * a.d.H * split * (a.d.E + 4), "partial");
  }
  launch_kept_attn_decode(
      ptr<bf16>(out), ptr<bf16>(q), ptr<bf16>(k_cache), ptr<bf16>(v_cache),
      block_tables.data_ptr<int>(), positions.data_ptr<long>(), a.turn,
      a.sink, split > 1 ? ptr<float>(*partial) : nullptr, rows,
      (int)block_tables.size(1), a.d.H, a.d.G, a.d.D, a.d.E, (int)window,
      (int)keep, (float)scale, bounded, q.stride(0), out.stride(0),
      (int)split, stream());
}

}  // namespace

void register_sublayer(pybind11::module_& m) {
  m.def("add_rms_next", &add_rms_next);
  m.def("experts_sum_next", &experts_sum_next);
  m.def("causal_conv", &causal_conv);
  m.def("clamped_glu", &clamped_glu);
  m.def("squared_relu", &squared_relu);
  m.def("norm_append", &norm_append);
  m.def("rope_norm_append", &rope_norm_append);
  m.def("kept_attn_fits", &kept_attn_fits);
  m.def("kept_attn_general", &kept_attn_general);
  m.def("kept_attn_prefill", &kept_attn_prefill);
  m.def("kept_attn_decode", &kept_attn_decode);
  m.def("sigmoid_attn_fits", &sigmoid_attn_fits);
  m.def("sigmoid_attn_general", &sigmoid_attn_general);
  m.def("sigmoid_attn_prefill", &sigmoid_attn_prefill);
  m.def("sigmoid_attn_decode", &sigmoid_attn_decode);
}
