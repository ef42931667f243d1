// torch op registrations of the heads library: softmax attention over paged caches of unequal key and value sizes, and what
// goes into them.
#include "torch_bindings.h"

namespace {

void head_attention(torch::Tensor& out, const torch::Tensor& q, const torch::Tensor& key_cache,
                    const torch::Tensor& value_cache, const torch::Tensor& block_tables, const torch::Tensor& seq_lens,
                    const torch::Tensor& query_start_loc, const std::optional<torch::Tensor>& gate, int64_t vdim,
                    double scale, double out_scale, int64_t max_query_len, int64_t max_seq_len, int64_t window,
                    int64_t min_query_len, int64_t chunk, int64_t keep_first, double softcap,
                    const std::optional<torch::Tensor>& sink, int64_t maps, double map_weight, double map_eps) {
  const char* op = "head_attention";
  LV_CHECK_DEVICE(q);
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(q));
  TORCH_CHECK(q.dim() == 3 && q.is_contiguous(), op, ": contiguous q [rows, heads, kpad]");
  const int64_t kv_heads = key_cache.size(1), rows = q.size(0), heads = q.size(1);
  const auto [kpad, vpad, bs] = head_cache_dims(key_cache, value_cache, kv_heads, q.scalar_type(), op);
  TORCH_CHECK(q.size(2) == kpad && vdim <= vpad, op, ": q and the caches disagree on the padded sizes");
  TORCH_CHECK(out.is_cuda() && out.dim() == 2 && out.stride(1) == 1 && out.size(0) == rows && out.size(1) == heads * vdim &&
                  out.scalar_type() == q.scalar_type(),
              op, ": out [rows, heads * vdim]");
  if (gate)
    TORCH_CHECK(gate->is_cuda() && gate->dim() == 2 && gate->stride(1) == 1 && gate->size(0) == rows &&
                    gate->size(1) == heads && gate->scalar_type() == q.scalar_type(),
                op, ": gate [rows, heads]");
  check_layout(query_start_loc, seq_lens, op);
  TORCH_CHECK(block_tables.is_cuda() && block_tables.dim() == 2 && block_tables.scalar_type() == at::kInt &&
                  block_tables.is_contiguous() && block_tables.size(0) >= seq_lens.numel(),
              op, ": block_tables int32 [num_seqs, blocks]");
  if (sink) check_f32(*sink, heads, op, "sink");
  const lvllm_head_options options{(int)window, (int)chunk, (int)keep_first, (int)maps, (int)min_query_len, (float)softcap,
                                   (float)map_weight, (float)map_eps, sink ? sink->data_ptr<float>() : nullptr};
  const int ns = (int)seq_lens.numel(), code = dtype_code(q, op);
  const int64_t need = lvllm_head_attention_workspace_bytes((int)rows, ns, (int)heads, (int)kv_heads, (int)kpad, (int)vpad,
                                                            (int)bs, (int)max_seq_len, &options, code);
  torch::Tensor ws;
  if (need > 0) ws = torch::empty({need}, q.options().dtype(at::kByte));
  check(lvllm_head_attention(out.data_ptr(), out.stride(0), q.data_ptr(), key_cache.data_ptr(), value_cache.data_ptr(),
                             gate ? gate->data_ptr() : nullptr, gate ? gate->stride(0) : 0, block_tables.data_ptr<int>(),
                             seq_lens.data_ptr<int>(), query_start_loc.data_ptr<int>(), ns, (int)rows, (int)heads,
                             (int)kv_heads, (int)kpad, (int)vpad, (int)vdim, (int)block_tables.size(1), (int)bs,
                             key_cache.size(0), (float)scale, (float)out_scale, key_cache.stride(0), value_cache.stride(0),
                             (int)max_query_len, (int)max_seq_len, &options, need > 0 ? ws.data_ptr() : nullptr, need, code,
                             current_stream(q)));
}

torch::Tensor qk_norm_cache(const torch::Tensor& q, const torch::Tensor& k, const torch::Tensor& v,
                            const torch::Tensor& q_weight, const torch::Tensor& k_weight, double eps, int64_t heads,
                            int64_t kv_heads, torch::Tensor& key_cache, torch::Tensor& value_cache,
                            const torch::Tensor& slot_mapping) {
  const char* op = "qk_norm_cache";
  LV_CHECK_DEVICE(q);
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(q));
  const int64_t rows = q.size(0), dim = q.size(1) / heads, vdim = v.size(1) / kv_heads;
  TORCH_CHECK(q.dim() == 2 && k.dim() == 2 && v.dim() == 2 && q.size(1) == heads * dim && k.size(1) == kv_heads * dim &&
                  v.size(1) == kv_heads * vdim && k.size(0) == rows && v.size(0) == rows && q.stride(1) == 1 &&
                  k.stride(1) == 1 && v.stride(1) == 1 && q.stride(0) == k.stride(0) && q.stride(0) == v.stride(0) &&
                  k.scalar_type() == q.scalar_type() && v.scalar_type() == q.scalar_type(),
              op, ": q [rows, heads * dim], k [rows, kv_heads * dim], v [rows, kv_heads * vdim] with one row stride");
  check_f32(q_weight, dim, op, "q_weight");
  check_f32(k_weight, dim, op, "k_weight");
  const auto [kpad, vpad, bs] = head_cache_dims(key_cache, value_cache, kv_heads, q.scalar_type(), op);
  check_slots(slot_mapping, rows, op);
  auto q_out = torch::empty({rows, heads, kpad}, q.options());
  check(lvllm_qk_norm_cache(q_out.data_ptr(), key_cache.data_ptr(), value_cache.data_ptr(), q.data_ptr(), k.data_ptr(),
                            v.data_ptr(), q.stride(0), q_weight.data_ptr<float>(), k_weight.data_ptr<float>(), (float)eps,
                            (int)rows, (int)heads, (int)kv_heads, (int)dim, (int)vdim, (int)kpad, (int)vpad,
                            slot_mapping.data_ptr<int64_t>(), key_cache.size(0), (int)bs, key_cache.stride(0),
                            value_cache.stride(0), dtype_code(q, op), current_stream(q)));
  return q_out;
}

// q [rows, heads * maps * dim], k [rows, kv_heads * maps * dim], v [rows, kv_heads * vdim] (k itself: the keys are the values)
torch::Tensor rotary_cache(const torch::Tensor& q, const torch::Tensor& k, const torch::Tensor& v,
                           const std::optional<torch::Tensor>& q_weight, const std::optional<torch::Tensor>& k_weight, double eps,
                           int64_t heads, int64_t kv_heads, int64_t maps, const torch::Tensor& positions,
                           const torch::Tensor& turns, torch::Tensor& key_cache, torch::Tensor& value_cache,
                           const torch::Tensor& slot_mapping) {
  const char* op = "rotary_cache";
  LV_CHECK_DEVICE(q);
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(q));
  TORCH_CHECK(heads > 0 && kv_heads > 0 && (maps == 1 || maps == 2), op, ": heads, kv_heads, one or two maps");
  const int64_t rows = q.size(0), dim = q.size(1) / (heads * maps), vdim = v.size(1) / kv_heads;
  check_rows2d(q, rows, heads * maps * dim, q.scalar_type(), op, "q");
  check_rows2d(k, rows, kv_heads * maps * dim, q.scalar_type(), op, "k");
  check_rows2d(v, rows, kv_heads * vdim, q.scalar_type(), op, "v");
  TORCH_CHECK(q.stride(0) == k.stride(0) && q.stride(0) == v.stride(0), op, ": one row stride");
  if (q_weight) check_f32(*q_weight, q.size(1), op, "q_weight");
  if (k_weight) check_f32(*k_weight, k.size(1), op, "k_weight");
  check_rot(positions, turns, rows, op);
  check_slots(slot_mapping, rows, op);
  const auto [kpad, vpad, bs] = head_cache_dims(key_cache, value_cache, kv_heads, q.scalar_type(), op);
  auto q_out = torch::empty({rows, heads, kpad}, q.options());
  check(lvllm_rotary_cache(q_out.data_ptr(), key_cache.data_ptr(), value_cache.data_ptr(), q.data_ptr(), k.data_ptr(),
                           v.data_ptr(), q.stride(0), q_weight ? q_weight->data_ptr<float>() : nullptr,
                           k_weight ? k_weight->data_ptr<float>() : nullptr, (float)eps, (int)rows, (int)heads, (int)kv_heads,
                           (int)maps, (int)dim, (int)vdim, (int)kpad, (int)vpad, positions.data_ptr<int64_t>(),
                           turns.data_ptr<double>(), (int)turns.numel() * 2, slot_mapping.data_ptr<int64_t>(),
                           key_cache.size(0), (int)bs, key_cache.stride(0), value_cache.stride(0), dtype_code(q, op),
                           current_stream(q)));
  return q_out;
}

}  // namespace

TORCH_LIBRARY_FRAGMENT(_C_amd, heads) {
  heads.def("head_attention(Tensor(a!) out, Tensor q, Tensor key_cache, Tensor value_cache, Tensor block_tables, "
             "Tensor seq_lens, Tensor query_start_loc, Tensor? gate, int vdim, float scale, float out_scale, "
             "int max_query_len, int max_seq_len, int window=0, int min_query_len=0, int chunk=0, int keep_first=0, "
             "float softcap=0., Tensor? sink=None, int maps=1, float map_weight=0., float map_eps=0.) -> ()");
  heads.impl("head_attention", torch::kCUDA, &head_attention);
  heads.def("qk_norm_cache(Tensor q, Tensor k, Tensor v, Tensor q_weight, Tensor k_weight, float eps, int heads, "
            "int kv_heads, Tensor(a!) key_cache, Tensor(b!) value_cache, Tensor slot_mapping) -> Tensor");
  heads.impl("qk_norm_cache", torch::kCUDA, &qk_norm_cache);
  heads.def("rotary_cache(Tensor q, Tensor k, Tensor v, Tensor? q_weight, Tensor? k_weight, float eps, int heads, int kv_heads, "
            "int maps, Tensor positions, Tensor turns, Tensor(a!) key_cache, Tensor(b!) value_cache, Tensor slot_mapping) "
            "-> Tensor");
  heads.impl("rotary_cache", torch::kCUDA, &rotary_cache);
}

PyMODINIT_FUNC PyInit__C_heads(void) {
  static struct PyModuleDef module = {PyModuleDef_HEAD_INIT, "_C_heads", nullptr, 0, nullptr};
  return PyModule_Create(&module);
}
