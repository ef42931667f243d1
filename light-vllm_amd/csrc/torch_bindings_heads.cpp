// torch op registrations of the heads library: softmax attention over paged caches of unequal key and value sizes.
#include "torch_bindings.h"

namespace {

void head_attention(torch::Tensor& out, const torch::Tensor& q, const torch::Tensor& key_cache,
                    const torch::Tensor& value_cache, const torch::Tensor& block_tables, const torch::Tensor& seq_lens,
                    const torch::Tensor& query_start_loc, const std::optional<torch::Tensor>& gate, int64_t vdim,
                    double scale, double out_scale, int64_t max_query_len, int64_t max_seq_len, int64_t window,
                    int64_t min_query_len) {
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
  const int ns = (int)seq_lens.numel(), code = dtype_code(q, op);
  const int64_t need = lvllm_head_attention_workspace_bytes((int)rows, ns, (int)heads, (int)kv_heads, (int)kpad, (int)vpad,
                                                            (int)bs, (int)max_seq_len, code);
  torch::Tensor ws;
  if (need > 0) ws = torch::empty({need}, q.options().dtype(at::kByte));
  check(lvllm_head_attention(out.data_ptr(), out.stride(0), q.data_ptr(), key_cache.data_ptr(), value_cache.data_ptr(),
                             gate ? gate->data_ptr() : nullptr, gate ? gate->stride(0) : 0, block_tables.data_ptr<int>(),
                             seq_lens.data_ptr<int>(), query_start_loc.data_ptr<int>(), ns, (int)rows, (int)heads,
                             (int)kv_heads, (int)kpad, (int)vpad, (int)vdim, (int)block_tables.size(1), (int)bs,
                             key_cache.size(0), (float)scale, (float)out_scale, key_cache.stride(0), value_cache.stride(0),
                             (int)max_query_len, (int)max_seq_len, (int)window, (int)min_query_len, need > 0 ? ws.data_ptr() : nullptr, need, code,
                             current_stream(q)));
}

}  // namespace

TORCH_LIBRARY_FRAGMENT(_C_amd, heads) {
  heads.def("head_attention(Tensor(a!) out, Tensor q, Tensor key_cache, Tensor value_cache, Tensor block_tables, "
             "Tensor seq_lens, Tensor query_start_loc, Tensor? gate, int vdim, float scale, float out_scale, "
             "int max_query_len, int max_seq_len, int window=0, int min_query_len=0) -> ()");
  heads.impl("head_attention", torch::kCUDA, &head_attention);
}

PyMODINIT_FUNC PyInit__C_heads(void) {
  static struct PyModuleDef module = {PyModuleDef_HEAD_INIT, "_C_heads", nullptr, 0, nullptr};
  return PyModule_Create(&module);
}
