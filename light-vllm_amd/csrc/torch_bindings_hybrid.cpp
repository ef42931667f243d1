// torch op registrations of the hybrid library: row-wise operators and recurrences of the hybrid decoders.
#include "torch_bindings.h"

namespace {

torch::Tensor add_dyt(torch::Tensor& x, const std::optional<torch::Tensor>& y, const torch::Tensor& alpha,
                      const torch::Tensor& weight, const torch::Tensor& bias, at::ScalarType dtype) {
  check_residual(x, "add_dyt");
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(x));
  check_f32(alpha, 1, "add_dyt", "alpha");
  check_f32(weight, x.size(1), "add_dyt", "weight");
  check_f32(bias, x.size(1), "add_dyt", "bias");
  const Addend a = addend_of(y, x, dtype, "add_dyt");
  auto h = torch::empty(x.sizes(), x.options().dtype(dtype));
  float* xp = x.data_ptr<float>();
  check(lvllm_add_dyt(y ? xp : nullptr, xp, a.y, a.partials, a.num, h.data_ptr(), alpha.data_ptr<float>(),
                      weight.data_ptr<float>(), bias.data_ptr<float>(), (int)x.size(0), (int)x.size(1),
                      dtype_code(h, "add_dyt"), current_stream(x)));
  return h;
}

std::tuple<torch::Tensor, torch::Tensor> add_dyt_shift_mix(
    const torch::Tensor& x, const std::optional<torch::Tensor>& y, const torch::Tensor& mu, const torch::Tensor& alpha,
    const torch::Tensor& weight, const torch::Tensor& bias, torch::Tensor& carried, const torch::Tensor& state_slots,
    const torch::Tensor& query_start_loc, const torch::Tensor& seq_lens, at::ScalarType dtype) {
  const char* op = "add_dyt_shift_mix";
  check_residual(x, op);
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(x));
  const int64_t rows = x.size(0), width = x.size(1);
  check_f32(alpha, 1, op, "alpha");
  check_f32(weight, width, op, "weight");
  check_f32(bias, width, op, "bias");
  TORCH_CHECK(mu.dim() == 2, op, ": mu must be [mixes, width]");
  check_f32(mu, mu.size(0) * width, op, "mu");
  check_layout(query_start_loc, seq_lens, op);
  check_state(carried, state_slots, width, seq_lens.numel(), op);
  const Addend a = addend_of(y, x, dtype, op);
  auto x_out = torch::empty(y ? x.sizes() : at::IntArrayRef({0, 0}), x.options());  // (nothing to add: x stays)
  auto mix = torch::empty({mu.size(0), rows, width}, x.options().dtype(dtype));
  check(lvllm_add_dyt_shift_mix(y ? x_out.data_ptr<float>() : nullptr, x.data_ptr<float>(), a.y, a.partials, a.num,
                                mix.data_ptr(), mu.data_ptr<float>(), (int)mu.size(0), alpha.data_ptr<float>(),
                                weight.data_ptr<float>(), bias.data_ptr<float>(), carried.data_ptr<float>(),
                                carried.stride(0), state_slots.data_ptr<int>(), (int)carried.size(0),
                                query_start_loc.data_ptr<int>(), seq_lens.data_ptr<int>(), (int)seq_lens.numel(),
                                (int)rows, (int)width, dtype_code(mix, op), current_stream(x)));
  return {x_out, mix};
}

void relu_squared(torch::Tensor& out, const torch::Tensor& x) {
  LV_CHECK_DEVICE(x);
  TORCH_CHECK(x.is_contiguous() && out.is_contiguous() && out.sizes() == x.sizes() && out.scalar_type() == x.scalar_type(),
              "relu_squared: contiguous tensors of one shape and dtype");
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(x));
  check(lvllm_relu_squared(out.data_ptr(), x.data_ptr(), x.numel(), dtype_code(x, "relu_squared"), current_stream(x)));
}

void head_norm_gate(torch::Tensor& out, const torch::Tensor& o, const torch::Tensor& gate, const torch::Tensor& weight,
                    double eps, double scale) {
  const char* op = "head_norm_gate";
  LV_CHECK_DEVICE(o);
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(o));
  TORCH_CHECK(o.dim() == 3 && o.is_contiguous() && o.scalar_type() == at::kFloat, op, ": o float32 [rows, heads, vdim]");
  const int64_t rows = o.size(0), heads = o.size(1), vdim = o.size(2);
  TORCH_CHECK(out.dim() == 2 && out.stride(1) == 1 && out.size(0) == rows && out.size(1) == heads * vdim &&
                  gate.dim() == 2 && gate.stride(1) == 1 && gate.size(0) == rows && gate.size(1) == heads * vdim &&
                  gate.scalar_type() == out.scalar_type(),
              op, ": out and gate [rows, heads * vdim]");
  const bool shared = weight.numel() == vdim;
  check_f32(weight, shared ? vdim : heads * vdim, op, "weight");
  check(lvllm_head_norm_gate(out.data_ptr(), out.stride(0), o.data_ptr<float>(), gate.data_ptr(), gate.stride(0),
                             weight.data_ptr<float>(), shared ? 0 : (int)vdim, (float)eps, (float)scale, (int)rows,
                             (int)heads, (int)vdim, dtype_code(out, op), current_stream(o)));
}

torch::Tensor log_decay(const torch::Tensor& u, const torch::Tensor& a_t, const torch::Tensor& bias, int64_t kind,
                        double inv_tau) {
  const char* op = "log_decay";
  LV_CHECK_DEVICE(u);
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(u));
  TORCH_CHECK(u.dim() == 2 && u.stride(1) == 1 && a_t.dim() == 2 && a_t.size(0) == u.size(1), op,
              ": u [rows, rank], a_t [rank, channels]");
  check_f32(a_t, a_t.size(0) * a_t.size(1), op, "a_t");
  check_f32(bias, a_t.size(1), op, "bias");
  auto out = torch::empty({u.size(0), a_t.size(1)}, u.options().dtype(at::kFloat));
  check(lvllm_log_decay(out.data_ptr<float>(), u.data_ptr(), u.stride(0), a_t.data_ptr<float>(), bias.data_ptr<float>(),
                        (int)kind, (float)inv_tau, (int)u.size(0), (int)u.size(1), (int)a_t.size(1), dtype_code(u, op),
                        current_stream(u)));
  return out;
}

torch::Tensor recurrent_scan(const torch::Tensor& q, const torch::Tensor& k, const torch::Tensor& v,
                             const torch::Tensor& log_decay, const std::optional<torch::Tensor>& bonus, double q_scale,
                             torch::Tensor& state, const torch::Tensor& state_slots, const torch::Tensor& query_start_loc,
                             const torch::Tensor& seq_lens) {
  const char* op = "recurrent_scan";
  LV_CHECK_DEVICE(q);
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(q));
  TORCH_CHECK(state.dim() == 4, op, ": state [slots, heads, dk, dv]");
  const int64_t rows = q.size(0), heads = state.size(1), dk = state.size(2), dv = state.size(3);
  TORCH_CHECK(q.dim() == 2 && k.dim() == 2 && v.dim() == 2 && q.size(1) == heads * dk && k.size(1) == heads * dk &&
                  v.size(1) == heads * dv && k.size(0) == rows && v.size(0) == rows && q.stride(1) == 1 &&
                  k.stride(1) == 1 && v.stride(1) == 1 && k.scalar_type() == q.scalar_type() &&
                  v.scalar_type() == q.scalar_type(),
              op, ": q, k [rows, heads * dk], v [rows, heads * dv]");
  check_f32(log_decay, rows * heads * dk, op, "log_decay");
  if (bonus) check_f32(*bonus, heads * dk, op, "bonus");
  check_layout(query_start_loc, seq_lens, op);
  check_state(state, state_slots, heads * dk * dv, seq_lens.numel(), op);
  auto o = torch::empty({rows, heads, dv}, q.options().dtype(at::kFloat));
  check(lvllm_recurrent_scan(o.data_ptr<float>(), q.data_ptr(), k.data_ptr(), v.data_ptr(), q.stride(0), k.stride(0),
                             v.stride(0), log_decay.data_ptr<float>(), bonus ? bonus->data_ptr<float>() : nullptr,
                             (float)q_scale, state.data_ptr<float>(), state.stride(0), state_slots.data_ptr<int>(),
                             (int)state.size(0), query_start_loc.data_ptr<int>(), seq_lens.data_ptr<int>(),
                             (int)seq_lens.numel(), (int)heads, (int)dk, (int)dv, dtype_code(q, op), current_stream(q)));
  return o;
}

void recurrent_mix(torch::Tensor& out, const torch::Tensor& q, const torch::Tensor& k, const torch::Tensor& v,
                   const torch::Tensor& u, const torch::Tensor& a_t, const torch::Tensor& decay_bias, int64_t kind,
                   double inv_tau, const std::optional<torch::Tensor>& bonus, double q_scale, const torch::Tensor& gate,
                   const torch::Tensor& norm_weight, double eps, double out_scale, torch::Tensor& state,
                   const torch::Tensor& state_slots, const torch::Tensor& query_start_loc, const torch::Tensor& seq_lens,
                   int64_t max_query_len) {
  const char* op = "recurrent_mix";
  LV_CHECK_DEVICE(q);
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(q));
  TORCH_CHECK(state.dim() == 4, op, ": state [slots, heads, dk, dv]");
  const int64_t rows = q.size(0), heads = state.size(1), dk = state.size(2), dv = state.size(3), rank = u.size(1);
  auto rows_of = [&](const torch::Tensor& t, int64_t cols, const char* what) {
    TORCH_CHECK(t.is_cuda() && t.dim() == 2 && t.size(0) == rows && t.size(1) == cols && t.stride(1) == 1 &&
                    t.scalar_type() == q.scalar_type(),
                op, ": ", what, " must be [rows, ", cols, "] of the compute dtype");
  };
  rows_of(q, heads * dk, "q");
  rows_of(k, heads * dk, "k");
  rows_of(v, heads * dv, "v");
  rows_of(u, rank, "u");
  rows_of(gate, heads * dv, "gate");
  rows_of(out, heads * dv, "out");
  TORCH_CHECK(a_t.dim() == 2 && a_t.size(0) == rank, op, ": a_t [rank, heads * dk]");
  check_f32(a_t, rank * heads * dk, op, "a_t");
  check_f32(decay_bias, heads * dk, op, "decay_bias");
  if (bonus) check_f32(*bonus, heads * dk, op, "bonus");
  const bool shared = norm_weight.numel() == dv;
  check_f32(norm_weight, shared ? dv : heads * dv, op, "norm_weight");
  check_layout(query_start_loc, seq_lens, op);
  check_state(state, state_slots, heads * dk * dv, seq_lens.numel(), op);
  const int ns = (int)seq_lens.numel();
  if (max_query_len <= 1) TORCH_CHECK(ns == rows, op, ": a step of single tokens has one row per sequence");
  const int64_t need = lvllm_recurrent_mix_workspace_bytes((int)rows, ns, (int)heads, (int)dk, (int)dv, (int)max_query_len);
  torch::Tensor ws;
  if (need > 0) ws = torch::empty({need}, q.options().dtype(at::kByte));
  check(lvllm_recurrent_mix(out.data_ptr(), out.stride(0), q.data_ptr(), k.data_ptr(), v.data_ptr(), q.stride(0),
                            k.stride(0), v.stride(0), u.data_ptr(), u.stride(0), a_t.data_ptr<float>(),
                            decay_bias.data_ptr<float>(), (int)rank, (int)kind, (float)inv_tau,
                            bonus ? bonus->data_ptr<float>() : nullptr, (float)q_scale, gate.data_ptr(), gate.stride(0),
                            norm_weight.data_ptr<float>(), shared ? 0 : (int)dv, (float)eps, (float)out_scale,
                            state.data_ptr<float>(), state.stride(0), state_slots.data_ptr<int>(), (int)state.size(0),
                            query_start_loc.data_ptr<int>(), seq_lens.data_ptr<int>(), ns, (int)rows, (int)heads, (int)dk,
                            (int)dv, (int)max_query_len, ws.defined() ? ws.data_ptr() : nullptr, need, dtype_code(q, op), current_stream(q)));
}

}  // namespace

TORCH_LIBRARY_FRAGMENT(_C_amd, hybrid) {
  hybrid.def("add_dyt(Tensor(a!) x, Tensor? y, Tensor alpha, Tensor weight, Tensor bias, ScalarType dtype) -> Tensor");
  hybrid.impl("add_dyt", torch::kCUDA, &add_dyt);
  hybrid.def("add_dyt_shift_mix(Tensor x, Tensor? y, Tensor mu, Tensor alpha, Tensor weight, Tensor bias, "
             "Tensor(a!) carried, Tensor state_slots, Tensor query_start_loc, Tensor seq_lens, ScalarType dtype) "
             "-> (Tensor, Tensor)");
  hybrid.impl("add_dyt_shift_mix", torch::kCUDA, &add_dyt_shift_mix);
  hybrid.def("relu_squared(Tensor(a!) out, Tensor x) -> ()");
  hybrid.impl("relu_squared", torch::kCUDA, &relu_squared);
  hybrid.def("recurrent_mix(Tensor(a!) out, Tensor q, Tensor k, Tensor v, Tensor u, Tensor a_t, Tensor decay_bias, "
             "int kind, float inv_tau, Tensor? bonus, float q_scale, Tensor gate, Tensor norm_weight, float eps, "
             "float out_scale, Tensor(b!) state, Tensor state_slots, Tensor query_start_loc, Tensor seq_lens, "
             "int max_query_len) -> ()");
  hybrid.impl("recurrent_mix", torch::kCUDA, &recurrent_mix);
  hybrid.def("head_norm_gate(Tensor(a!) out, Tensor o, Tensor gate, Tensor weight, float eps, float scale) -> ()");
  hybrid.impl("head_norm_gate", torch::kCUDA, &head_norm_gate);
  hybrid.def("log_decay(Tensor u, Tensor a_t, Tensor bias, int kind, float inv_tau) -> Tensor");
  hybrid.impl("log_decay", torch::kCUDA, &log_decay);
  hybrid.def("recurrent_scan(Tensor q, Tensor k, Tensor v, Tensor log_decay, Tensor? bonus, float q_scale, "
             "Tensor(a!) state, Tensor state_slots, Tensor query_start_loc, Tensor seq_lens) -> Tensor");
  hybrid.impl("recurrent_scan", torch::kCUDA, &recurrent_scan);
}

PyMODINIT_FUNC PyInit__C_hybrid(void) {
  static struct PyModuleDef module = {PyModuleDef_HEAD_INIT, "_C_hybrid", nullptr, 0, nullptr};
  return PyModule_Create(&module);
}
