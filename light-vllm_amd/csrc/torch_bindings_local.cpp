// torch op registrations of the local library: retention, norms around sublayers, the embedding with a table of token pairs.
#include "torch_bindings.h"

namespace {

void retention(torch::Tensor& out, const torch::Tensor& q, const torch::Tensor& k, const torch::Tensor& v,
               const torch::Tensor& positions, const torch::Tensor& turns, const torch::Tensor& head_decay, double q_scale,
               const torch::Tensor& gate, const std::optional<torch::Tensor>& norm_weight, double eps, double out_scale,
               torch::Tensor& state, const torch::Tensor& state_slots, const torch::Tensor& query_start_loc,
               const torch::Tensor& seq_lens, int64_t max_query_len) {
  const char* op = "retention";
  LV_CHECK_DEVICE(q);
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(q));
  TORCH_CHECK(state.dim() == 4, op, ": state [slots, heads, dk, dv]");
  const int64_t rows = q.size(0), heads = state.size(1), dk = state.size(2), dv = state.size(3);
  check_rows2d(q, rows, heads * dk, q.scalar_type(), op, "q");
  check_rows2d(k, rows, heads * dk, q.scalar_type(), op, "k");
  check_rows2d(v, rows, heads * dv, q.scalar_type(), op, "v");
  check_rows2d(gate, rows, heads * dv, q.scalar_type(), op, "gate");
  check_rows2d(out, rows, heads * dv, q.scalar_type(), op, "out");
  check_rot(positions, turns, rows, op);
  check_f32(head_decay, 2 * heads, op, "head_decay");
  const bool shared = norm_weight && norm_weight->numel() == dv;
  if (norm_weight) check_f32(*norm_weight, shared ? dv : heads * dv, op, "norm_weight");
  check_layout(query_start_loc, seq_lens, op);
  check_state(state, state_slots, heads * dk * dv, seq_lens.numel(), op);
  const int ns = (int)seq_lens.numel();
  if (max_query_len <= 1) TORCH_CHECK(ns == rows, op, ": a step of single tokens has one row per sequence");
  const int64_t need = lvllm_retention_workspace_bytes((int)rows, ns, (int)heads, (int)dk, (int)dv, (int)max_query_len);
  torch::Tensor ws;
  if (need > 0) ws = torch::empty({need}, q.options().dtype(at::kByte));
  check(lvllm_retention(out.data_ptr(), out.stride(0), q.data_ptr(), k.data_ptr(), v.data_ptr(), q.stride(0), k.stride(0),
                        v.stride(0), positions.data_ptr<int64_t>(), turns.data_ptr<double>(), (int)turns.numel() * 2,
                        head_decay.data_ptr<float>(), (float)q_scale, gate.data_ptr(), gate.stride(0),
                        norm_weight ? norm_weight->data_ptr<float>() : nullptr, shared ? 0 : (int)dv, (float)eps,
                        (float)out_scale, state.data_ptr<float>(), state.stride(0), state_slots.data_ptr<int>(),
                        (int)state.size(0), query_start_loc.data_ptr<int>(), seq_lens.data_ptr<int>(), ns, (int)rows, (int)heads,
                        (int)dk, (int)dv, (int)max_query_len, ws.defined() ? ws.data_ptr() : nullptr, need, dtype_code(q, op),
                        current_stream(q)));
}

// y: rows of the compute dtype, fp32 slabs [s, rows, width], or (with slots [rows, n]) the slots of a mixture; a second branch
// `other` makes the sublayer's output half the sum of both branches' norms
torch::Tensor sandwich_norm(torch::Tensor& x, const torch::Tensor& y, const std::optional<torch::Tensor>& slots,
                            const std::optional<torch::Tensor>& bias, const std::optional<torch::Tensor>& y_weight,
                            const std::optional<torch::Tensor>& other, const std::optional<torch::Tensor>& other_bias,
                            const std::optional<torch::Tensor>& other_weight, const torch::Tensor& weight,
                            const torch::Tensor& next_weight, double eps, at::ScalarType dtype) {
  const char* op = "sandwich_norm";
  check_residual(x, op);
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(x));
  const int64_t rows = x.size(0), width = x.size(1);
  check_f32(weight, width, op, "weight");
  check_f32(next_weight, width, op, "next_weight");
  lvllm_sandwich_branch branches[2] = {};
  auto fill = [&](lvllm_sandwich_branch& r, const torch::Tensor& t, const std::optional<torch::Tensor>& b,
                  const std::optional<torch::Tensor>& w, const std::optional<torch::Tensor>& s) {
    if (s) {
      TORCH_CHECK(s->dim() == 2 && s->size(0) == rows && t.is_cuda() && t.dim() == 2 && t.is_contiguous() &&
                      t.size(1) == width && t.scalar_type() == dtype,
                  op, ": slots int32 [rows, n] of y [slots, width]");
      check_i32(*s, s->numel(), op, "slots");
      r.y = t.data_ptr();
      r.slots = s->data_ptr<int>();
      r.num_slots = (int)s->size(1);
      r.total_slots = (int)t.size(0);
    } else {
      const Addend a = addend_of(t, x, dtype, op);
      r.y = a.y;
      r.partials = a.partials;
      r.num_partials = a.num;
    }
    if (b) {
      check_f32(*b, width, op, "bias");
      r.bias = b->data_ptr<float>();
    }
    if (w) {
      check_f32(*w, width, op, "a branch's weight");
      r.weight = w->data_ptr<float>();
    }
  };
  fill(branches[0], y, bias, y_weight, slots);
  if (other) fill(branches[1], *other, other_bias, other_weight, std::nullopt);
  auto h = torch::empty(x.sizes(), x.options().dtype(dtype));
  check(lvllm_sandwich_norm(x.data_ptr<float>(), h.data_ptr(), branches, other ? 2 : 1, weight.data_ptr<float>(),
                            next_weight.data_ptr<float>(), (float)eps, (int)rows, (int)width, dtype_code(h, op),
                            current_stream(x)));
  return h;
}

torch::Tensor pair_embed(torch::Tensor& x, const torch::Tensor& table, const std::optional<torch::Tensor>& pairs,
                         const torch::Tensor& ids, torch::Tensor& previous, const torch::Tensor& state_slots,
                         const torch::Tensor& query_start_loc, const torch::Tensor& seq_lens, int64_t mul_previous,
                         int64_t mul_current, const torch::Tensor& weight, double eps) {
  const char* op = "pair_embed";
  check_residual(x, op);
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(x));
  const int64_t rows = x.size(0), width = x.size(1);
  TORCH_CHECK(table.is_cuda() && table.dim() == 2 && table.is_contiguous() && table.size(1) == width && ids.is_cuda() &&
                  ids.scalar_type() == at::kLong && ids.is_contiguous() && ids.numel() == rows,
              op, ": table [vocab, width], ids int64 [rows]");
  if (pairs)
    TORCH_CHECK(pairs->is_cuda() && pairs->dim() == 2 && pairs->is_contiguous() && pairs->size(1) == width &&
                    pairs->size(0) >= 2 && pairs->scalar_type() == table.scalar_type(),
                op, ": pairs [buckets + 1, width]");
  check_layout(query_start_loc, seq_lens, op);
  check_i32(previous, 1, op, "previous");
  check_i32(state_slots, seq_lens.numel(), op, "state_slots");
  check_f32(weight, width, op, "weight");
  auto h = torch::empty(x.sizes(), table.options());
  check(lvllm_pair_embed(x.data_ptr<float>(), h.data_ptr(), table.data_ptr(), pairs ? pairs->data_ptr() : nullptr,
                         ids.data_ptr<int64_t>(), previous.data_ptr<int>(), state_slots.data_ptr<int>(), (int)previous.numel(),
                         query_start_loc.data_ptr<int>(), seq_lens.data_ptr<int>(), (int)seq_lens.numel(), mul_previous,
                         mul_current, pairs ? (int)pairs->size(0) - 1 : 0, weight.data_ptr<float>(), (float)eps, (int)rows,
                         (int)table.size(0), (int)width, dtype_code(table, op), current_stream(x)));
  return h;
}

}  // namespace

TORCH_LIBRARY_FRAGMENT(_C_amd, local) {
  local.def("retention(Tensor(a!) out, Tensor q, Tensor k, Tensor v, Tensor positions, Tensor turns, Tensor head_decay, "
            "float q_scale, Tensor gate, Tensor? norm_weight, float eps, float out_scale, Tensor(b!) state, "
            "Tensor state_slots, Tensor query_start_loc, Tensor seq_lens, int max_query_len) -> ()");
  local.impl("retention", torch::kCUDA, &retention);
  local.def("sandwich_norm(Tensor(a!) x, Tensor y, Tensor? slots, Tensor? bias, Tensor? y_weight, Tensor? other, "
            "Tensor? other_bias, Tensor? other_weight, Tensor weight, Tensor next_weight, float eps, ScalarType dtype) -> Tensor");
  local.impl("sandwich_norm", torch::kCUDA, &sandwich_norm);
  local.def("pair_embed(Tensor(a!) x, Tensor table, Tensor? pairs, Tensor ids, Tensor(b!) previous, Tensor state_slots, "
            "Tensor query_start_loc, Tensor seq_lens, int mul_previous, int mul_current, Tensor weight, float eps) -> Tensor");
  local.impl("pair_embed", torch::kCUDA, &pair_embed);
}

PyMODINIT_FUNC PyInit__C_local(void) {
  static struct PyModuleDef module = {PyModuleDef_HEAD_INIT, "_C_local", nullptr, 0, nullptr};
  return PyModule_Create(&module);
}
