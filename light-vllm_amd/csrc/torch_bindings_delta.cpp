// torch op registrations of the delta library: residual streams, short convolutions, the gated delta rule.
#include <cmath>

#include "torch_bindings.h"

namespace {

// x_in [streams, rows, width] (a stream stride of 0: one row serves all); y: rows of the compute dtype, fp32 slabs, or the slots
// of a mixture with their weights
torch::Tensor stream_mix(const std::optional<torch::Tensor>& x_out, const torch::Tensor& x_in, const torch::Tensor& y,
                         const std::optional<torch::Tensor>& slots, const std::optional<torch::Tensor>& slot_weights,
                         const torch::Tensor& mix, const torch::Tensor& out, const torch::Tensor& in, const torch::Tensor& weight,
                         double eps, at::ScalarType dtype) {
  const char* op = "stream_mix";
  auto streams_ok = [](const torch::Tensor& t) {
    return t.is_cuda() && t.dim() == 3 && t.scalar_type() == at::kFloat && (t.numel() == 0 || t[0].is_contiguous());
  };
  TORCH_CHECK(streams_ok(x_in), op, ": streams float32 [n, rows, width], each contiguous");
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(x_in));
  const int64_t n = x_in.size(0), rows = x_in.size(1), width = x_in.size(2);
  TORCH_CHECK(!x_out || (streams_ok(*x_out) && x_out->sizes() == x_in.sizes() && (n == 1 || x_out->stride(0) >= rows * width)), op,
              ": x_out of the streams' shape");
  check_f32(mix, n * n, op, "mix");
  check_f32(out, n, op, "out");
  check_f32(in, n, op, "in");
  check_f32(weight, width, op, "weight");
  Addend a;
  int per_row = 0, total = 0;
  if (slots) {
    TORCH_CHECK(slot_weights && slots->dim() == 2 && slots->size(0) == rows && y.is_cuda() && y.dim() == 2 && y.is_contiguous() &&
                    y.size(1) == width && y.scalar_type() == dtype,
                op, ": slots int32 [rows, n] of y [slots, width], with their weights");
    check_i32(*slots, slots->numel(), op, "slots");
    check_f32(*slot_weights, slots->numel(), op, "slot_weights");
    a.y = y.data_ptr();
    per_row = (int)slots->size(1);
    total = (int)y.size(0);
  } else {
    a = addend_of(y, x_in.select(0, 0), dtype, op);
  }
  auto h = torch::empty({rows, width}, x_in.options().dtype(dtype));
  check(lvllm_stream_mix(x_out ? x_out->data_ptr<float>() : nullptr, x_out ? x_out->stride(0) : 0, x_in.data_ptr<float>(),
                         x_in.stride(0), h.data_ptr(), a.y, a.partials, a.num, slots ? slots->data_ptr<int>() : nullptr,
                         slots ? slot_weights->data_ptr<float>() : nullptr, per_row, total, mix.data_ptr<float>(),
                         out.data_ptr<float>(), in.data_ptr<float>(), (int)n, weight.data_ptr<float>(), (float)eps, (int)rows,
                         (int)width, dtype_code(h, op), current_stream(x_in)));
  return h;
}

torch::Tensor stream_embed(torch::Tensor& x, const torch::Tensor& table, const torch::Tensor& ids, const torch::Tensor& in,
                           const torch::Tensor& weight, double eps) {
  const char* op = "stream_embed";
  check_residual(x, op);
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(x));
  TORCH_CHECK(table.is_cuda() && table.dim() == 2 && table.is_contiguous() && table.size(1) == x.size(1) && ids.is_cuda() &&
                  ids.scalar_type() == at::kLong && ids.is_contiguous() && ids.numel() == x.size(0),
              op, ": table [vocab, width], ids int64 [rows]");
  check_f32(in, in.numel(), op, "in");
  check_f32(weight, x.size(1), op, "weight");
  auto h = torch::empty(x.sizes(), table.options());
  check(lvllm_stream_embed(x.data_ptr<float>(), h.data_ptr(), table.data_ptr(), ids.data_ptr<int64_t>(), in.data_ptr<float>(),
                           (int)in.numel(), weight.data_ptr<float>(), (float)eps, (int)x.size(0), (int)table.size(0),
                           (int)x.size(1), dtype_code(table, op), current_stream(x)));
  return h;
}

torch::Tensor short_conv(const torch::Tensor& x, const torch::Tensor& weight, torch::Tensor& state,
                         const torch::Tensor& state_slots, const torch::Tensor& query_start_loc, const torch::Tensor& seq_lens,
                         int64_t max_query_len) {
  const char* op = "short_conv";
  LV_CHECK_DEVICE(x);
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(x));
  TORCH_CHECK(weight.dim() == 2 && x.dim() == 2, op, ": x [rows, channels], weight [taps, channels]");
  const int64_t rows = x.size(0), taps = weight.size(0), channels = weight.size(1);
  check_rows2d(x, rows, channels, x.scalar_type(), op, "x");
  check_f32(weight, taps * channels, op, "weight");
  check_layout(query_start_loc, seq_lens, op);
  check_state(state, state_slots, taps * channels, seq_lens.numel(), op);
  auto y = torch::empty({rows, channels}, x.options());
  check(lvllm_short_conv(y.data_ptr(), y.stride(0), x.data_ptr(), x.stride(0), weight.data_ptr<float>(), (int)taps,
                         (int)channels, state.data_ptr<float>(), state.stride(0), state_slots.data_ptr<int>(),
                         (int)state.size(0), query_start_loc.data_ptr<int>(), seq_lens.data_ptr<int>(), (int)seq_lens.numel(),
                         (int)max_query_len, dtype_code(x, op), current_stream(x)));
  return y;
}

struct DeltaShapes {
  lvllm_delta_sizes sizes;
  int64_t rows, heads, dk, dv;
};
// `cols` columns of q | k | v, heads and sizes from the state
DeltaShapes delta_shapes(const torch::Tensor& x, const torch::Tensor& state, int64_t kv_heads, int64_t k_at, int64_t v_at,
                         const torch::Tensor& out, const torch::Tensor& scale, const torch::Tensor& bias, const torch::Tensor& norm,
                         const torch::Tensor& beta, const char* op) {
  LV_CHECK_DEVICE(x);
  TORCH_CHECK(state.dim() == 4 && kv_heads > 0 && state.size(1) % kv_heads == 0, op,
              ": state [slots, heads, dk, dv], heads a multiple of kv_heads");
  const int64_t rows = x.size(0), heads = state.size(1), dk = state.size(2), dv = state.size(3);
  TORCH_CHECK(x.dim() == 2 && x.stride(1) == 1 && k_at >= kv_heads * dk && v_at >= k_at + kv_heads * dk &&
                  x.size(1) >= v_at + heads * dv,
              op, ": q [rows, kv_heads * dk], k at column k_at, v [rows, heads * dv] at column v_at");
  check_rows2d(out, rows, heads * dv, x.scalar_type(), op, "out");
  check_rows2d(beta, rows, heads, x.scalar_type(), op, "beta");
  check_f32(scale, heads * dk, op, "decay_scale");
  check_f32(bias, heads * dk, op, "decay_bias");
  check_f32(norm, dv, op, "norm_weight");
  return {{(int)heads, (int)kv_heads, (int)dk, (int)dv, (int)k_at, (int)v_at, 1.f / std::sqrt((float)dk)}, rows, heads, dk, dv};
}

void delta_step(torch::Tensor& out, const torch::Tensor& x, int64_t kv_heads, int64_t k_at, int64_t v_at, const torch::Tensor& u,
                const torch::Tensor& z, const torch::Tensor& beta, const torch::Tensor& conv_weight, torch::Tensor& conv_state,
                const torch::Tensor& decay_w, const torch::Tensor& gate_w, const torch::Tensor& decay_scale,
                const torch::Tensor& decay_bias, const torch::Tensor& norm_weight, double eps, torch::Tensor& state,
                const torch::Tensor& state_slots, const torch::Tensor& seq_lens) {
  const char* op = "delta_step";
  const DeltaShapes d = delta_shapes(x, state, kv_heads, k_at, v_at, out, decay_scale, decay_bias, norm_weight, beta, op);
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(x));
  const int64_t ns = seq_lens.numel(), piece = 16 / x.element_size();
  check_i32(seq_lens, ns, op, "seq_lens");
  TORCH_CHECK(ns == d.rows, op, ": one row per sequence");
  check_rows2d(u, d.rows, u.size(1), x.scalar_type(), op, "u");
  check_rows2d(z, d.rows, z.size(1), x.scalar_type(), op, "z");
  TORCH_CHECK(u.stride(0) == x.stride(0) && z.stride(0) == x.stride(0) && beta.stride(0) == x.stride(0), op, ": one row stride");
  auto low_rank = [&](const torch::Tensor& w, int64_t rank, int64_t cols, const char* what) {
    TORCH_CHECK(w.is_cuda() && w.is_contiguous() && w.dim() == 3 && w.scalar_type() == x.scalar_type() &&
                    w.size(0) == (rank + piece - 1) / piece && w.size(1) == cols && w.size(2) == piece,
                op, ": ", what, " [pieces of the rank, ", cols, ", ", piece, "]");
  };
  low_rank(decay_w, u.size(1), d.heads * d.dk, "decay_w");
  low_rank(gate_w, z.size(1), d.heads * d.dv, "gate_w");
  TORCH_CHECK(conv_weight.dim() == 2, op, ": conv_weight [taps, channels]");
  const int64_t taps = conv_weight.size(0), channels = conv_weight.size(1);
  TORCH_CHECK(channels <= x.size(1) && channels >= v_at + d.heads * d.dv, op, ": a convolution for every channel of q, k and v");
  check_f32(conv_weight, taps * channels, op, "conv_weight");
  check_state(conv_state, state_slots, taps * channels, ns, op);
  check_state(state, state_slots, d.heads * d.dk * d.dv, ns, op);
  TORCH_CHECK(conv_state.size(0) == state.size(0), op, ": both states have the same slots");
  check(lvllm_delta_step(out.data_ptr(), out.stride(0), x.data_ptr(), x.stride(0), u.data_ptr(), z.data_ptr(), beta.data_ptr(),
                         conv_weight.data_ptr<float>(), (int)taps, (int)channels, conv_state.data_ptr<float>(),
                         conv_state.stride(0), decay_w.data_ptr(), (int)u.size(1), gate_w.data_ptr(), (int)z.size(1),
                         decay_scale.data_ptr<float>(), decay_bias.data_ptr<float>(), norm_weight.data_ptr<float>(), (float)eps,
                         &d.sizes, state.data_ptr<float>(), state.stride(0), state_slots.data_ptr<int>(), (int)state.size(0),
                         seq_lens.data_ptr<int>(), (int)ns, dtype_code(x, op), current_stream(x)));
}

void delta_chunks(torch::Tensor& out, const torch::Tensor& y, int64_t kv_heads, int64_t k_at, int64_t v_at, const torch::Tensor& u,
                  const torch::Tensor& beta, const torch::Tensor& a_t, const torch::Tensor& decay_scale,
                  const torch::Tensor& decay_bias, const torch::Tensor& gate, const torch::Tensor& norm_weight, double eps,
                  torch::Tensor& state, const torch::Tensor& state_slots, const torch::Tensor& query_start_loc,
                  const torch::Tensor& seq_lens, int64_t max_query_len) {
  const char* op = "delta_chunks";
  const DeltaShapes d = delta_shapes(y, state, kv_heads, k_at, v_at, out, decay_scale, decay_bias, norm_weight, beta, op);
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(y));
  const int64_t ns = seq_lens.numel();
  check_rows2d(u, d.rows, a_t.size(0), y.scalar_type(), op, "u");
  check_rows2d(gate, d.rows, d.heads * d.dv, y.scalar_type(), op, "gate");
  TORCH_CHECK(u.stride(0) == beta.stride(0) && a_t.dim() == 2, op, ": u and beta of one row stride, a_t [rank, heads * dk]");
  check_f32(a_t, u.size(1) * d.heads * d.dk, op, "a_t");
  check_layout(query_start_loc, seq_lens, op);
  check_state(state, state_slots, d.heads * d.dk * d.dv, ns, op);
  const int64_t need = lvllm_delta_chunks_workspace_bytes(&d.sizes, (int)d.rows, (int)ns);
  auto ws = torch::empty({need}, y.options().dtype(at::kByte));
  check(lvllm_delta_chunks(out.data_ptr(), out.stride(0), y.data_ptr(), y.stride(0), u.data_ptr(), beta.data_ptr(), u.stride(0),
                           a_t.data_ptr<float>(), (int)u.size(1), decay_scale.data_ptr<float>(), decay_bias.data_ptr<float>(),
                           gate.data_ptr(), gate.stride(0), norm_weight.data_ptr<float>(), (float)eps, &d.sizes,
                           state.data_ptr<float>(), state.stride(0), state_slots.data_ptr<int>(), (int)state.size(0),
                           query_start_loc.data_ptr<int>(), seq_lens.data_ptr<int>(), (int)ns, (int)d.rows, (int)max_query_len,
                           ws.data_ptr(), need, dtype_code(y, op), current_stream(y)));
}

}  // namespace

TORCH_LIBRARY_FRAGMENT(_C_amd, delta) {
  delta.def("stream_mix(Tensor(a!)? x_out, Tensor x_in, Tensor y, Tensor? slots, Tensor? slot_weights, Tensor mix, Tensor out, "
            "Tensor in_weights, Tensor weight, float eps, ScalarType dtype) -> Tensor");
  delta.impl("stream_mix", torch::kCUDA, &stream_mix);
  delta.def("stream_embed(Tensor(a!) x, Tensor table, Tensor ids, Tensor in_weights, Tensor weight, float eps) -> Tensor");
  delta.impl("stream_embed", torch::kCUDA, &stream_embed);
  delta.def("short_conv(Tensor x, Tensor weight, Tensor(a!) state, Tensor state_slots, Tensor query_start_loc, Tensor seq_lens, "
            "int max_query_len) -> Tensor");
  delta.impl("short_conv", torch::kCUDA, &short_conv);
  delta.def("delta_step(Tensor(a!) out, Tensor x, int kv_heads, int k_at, int v_at, Tensor u, Tensor z, Tensor beta, "
            "Tensor conv_weight, Tensor(b!) conv_state, Tensor decay_w, Tensor gate_w, Tensor decay_scale, Tensor decay_bias, "
            "Tensor norm_weight, float eps, Tensor(c!) state, Tensor state_slots, Tensor seq_lens) -> ()");
  delta.impl("delta_step", torch::kCUDA, &delta_step);
  delta.def("delta_chunks(Tensor(a!) out, Tensor y, int kv_heads, int k_at, int v_at, Tensor u, Tensor beta, Tensor a_t, "
            "Tensor decay_scale, Tensor decay_bias, Tensor gate, Tensor norm_weight, float eps, Tensor(b!) state, "
            "Tensor state_slots, Tensor query_start_loc, Tensor seq_lens, int max_query_len) -> ()");
  delta.impl("delta_chunks", torch::kCUDA, &delta_chunks);
}

PyMODINIT_FUNC PyInit__C_delta(void) {
  static struct PyModuleDef module = {PyModuleDef_HEAD_INIT, "_C_delta", nullptr, 0, nullptr};
  return PyModule_Create(&module);
}
