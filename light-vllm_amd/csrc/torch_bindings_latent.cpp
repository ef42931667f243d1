// torch op registrations of the latent library: latent attention, norms on sublayer outputs with depth averages.
#include "torch_bindings.h"

namespace {

void check_latent_rows(const torch::Tensor& cache, int64_t cpad, int64_t rpad, const char* op) {
  TORCH_CHECK(cache.is_cuda() && cache.dim() == 3 && cache.size(2) == cpad + rpad && blocks_are_dense(cache), op,
              ": cache [blocks, block_size, cpad + rpad], blocks dense");
}
void latent_cache(torch::Tensor& cache, const torch::Tensor& kv, const torch::Tensor& weight, double eps, int64_t cpad,
                  const torch::Tensor& positions, const torch::Tensor& turns, const torch::Tensor& slot_mapping, double grow) {
  const char* op = "latent_cache";
  LV_CHECK_DEVICE(kv);
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(kv));
  const int64_t rows = kv.size(0), rank = weight.numel(), rpad = cache.size(2) - cpad;
  check_latent_rows(cache, cpad, rpad, op);
  check_rows2d(kv, rows, kv.size(1), cache.scalar_type(), op, "kv");
  check_f32(weight, rank, op, "weight");
  check_rot(positions, turns, rows, op);
  TORCH_CHECK(kv.size(1) >= rank && slot_mapping.is_cuda() && slot_mapping.scalar_type() == at::kLong &&
                  slot_mapping.is_contiguous() && slot_mapping.numel() >= rows,
              op, ": slot_mapping int64 [rows]");
  check(lvllm_latent_cache(cache.data_ptr(), cache.stride(0), cache.size(0), (int)cache.size(1), (int)cpad, (int)rpad,
                           kv.data_ptr(), kv.stride(0), (int)rank, (int)(kv.size(1) - rank), weight.data_ptr<float>(),
                           (float)eps, positions.data_ptr<int64_t>(), turns.data_ptr<double>(), (int)turns.numel() * 2,
                           (float)grow, slot_mapping.data_ptr<int64_t>(), (int)rows, dtype_code(kv, op), current_stream(kv)));
}

// q [rows, q_rank] -> its RMS norm, [rows, q_pad]; the rows' cache entries as latent_cache writes them
torch::Tensor latent_down(const torch::Tensor& q, const torch::Tensor& q_weight, int64_t q_pad, torch::Tensor& cache,
                          const torch::Tensor& kv, const torch::Tensor& weight, double eps, int64_t cpad,
                          const torch::Tensor& positions, const torch::Tensor& turns, const torch::Tensor& slot_mapping,
                          double grow) {
  const char* op = "latent_down";
  LV_CHECK_DEVICE(q);
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(q));
  const int64_t rows = q.size(0), q_rank = q_weight.numel(), rank = weight.numel(), rpad = cache.size(2) - cpad;
  check_latent_rows(cache, cpad, rpad, op);
  check_rows2d(q, rows, q_rank, cache.scalar_type(), op, "q");
  check_rows2d(kv, rows, kv.size(1), cache.scalar_type(), op, "kv");
  check_f32(q_weight, q_rank, op, "q_weight");
  check_f32(weight, rank, op, "weight");
  check_rot(positions, turns, rows, op);
  check_slots(slot_mapping, rows, op);
  TORCH_CHECK(kv.size(1) >= rank, op, ": kv [rows, kv_rank + rot_dim]");
  auto out = torch::empty({rows, q_pad}, q.options());
  check(lvllm_latent_down(out.data_ptr(), q.data_ptr(), q.stride(0), (int)q_rank, (int)q_pad, q_weight.data_ptr<float>(),
                          cache.data_ptr(), cache.stride(0), cache.size(0), (int)cache.size(1), (int)cpad, (int)rpad,
                          kv.data_ptr(), kv.stride(0), (int)rank, (int)(kv.size(1) - rank), weight.data_ptr<float>(),
                          (float)eps, positions.data_ptr<int64_t>(), turns.data_ptr<double>(), (int)turns.numel() * 2,
                          (float)grow, slot_mapping.data_ptr<int64_t>(), (int)rows, dtype_code(q, op), current_stream(q)));
  return out;
}

// kv, weight, slot_mapping: the rows' own latents, written to the cache by the same launch
torch::Tensor latent_query(const torch::Tensor& q, const torch::Tensor& uk_t, int64_t dim, const torch::Tensor& positions,
                           const torch::Tensor& turns, const torch::Tensor& query_start_loc, int64_t absorbed_max,
                           torch::Tensor& cache, const std::optional<torch::Tensor>& kv,
                           const std::optional<torch::Tensor>& weight, double eps, const torch::Tensor& slot_mapping, double grow) {
  const char* op = "latent_query";
  LV_CHECK_DEVICE(q);
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(q));
  TORCH_CHECK(uk_t.is_cuda() && uk_t.dim() == 3 && uk_t.is_contiguous() && uk_t.scalar_type() == q.scalar_type() &&
                  cache.scalar_type() == q.scalar_type(),
              op, ": uk_t [heads, cpad, dpad]");
  const int64_t rows = q.size(0), heads = uk_t.size(0), cpad = uk_t.size(1), rpad = cache.size(2) - cpad;
  check_latent_rows(cache, cpad, rpad, op);
  TORCH_CHECK(q.dim() == 2 && q.size(1) % heads == 0 && q.size(1) / heads >= dim, op, ": q [rows, heads * (dim + rot_dim)]");
  check_rows2d(q, rows, q.size(1), q.scalar_type(), op, "q");
  check_rot(positions, turns, rows, op);
  check_i32(query_start_loc, 1, op, "query_start_loc");
  const int64_t rot_dim = q.size(1) / heads - dim;
  if (kv) {
    TORCH_CHECK(weight.has_value(), op, ": kv needs its norm's weight");
    check_rows2d(*kv, rows, weight->numel() + rot_dim, q.scalar_type(), op, "kv");
    check_f32(*weight, weight->numel(), op, "weight");
    TORCH_CHECK(slot_mapping.is_cuda() && slot_mapping.scalar_type() == at::kLong && slot_mapping.is_contiguous() &&
                    slot_mapping.numel() >= rows,
                op, ": slot_mapping int64 [rows]");
  }
  auto out = torch::empty({rows, heads, cpad + rpad}, q.options());
  check(lvllm_latent_query(out.data_ptr(), q.data_ptr(), q.stride(0), uk_t.data_ptr(), (int)heads, (int)dim,
                           (int)uk_t.size(2), (int)cpad, (int)rpad, (int)rot_dim, (int)turns.numel() * 2,
                           positions.data_ptr<int64_t>(), turns.data_ptr<double>(), (float)grow, query_start_loc.data_ptr<int>(),
                           (int)query_start_loc.numel() - 1, (int)absorbed_max, cache.data_ptr(), cache.stride(0),
                           cache.size(0), (int)cache.size(1), kv ? kv->data_ptr() : nullptr, kv ? kv->stride(0) : 0,
                           kv ? (int)weight->numel() : 0, kv ? weight->data_ptr<float>() : nullptr, (float)eps,
                           slot_mapping.data_ptr<int64_t>(), (int)rows, dtype_code(q, op), current_stream(q)));
  return out;
}

void latent_attention(torch::Tensor& out, const torch::Tensor& q, const torch::Tensor& cache, const torch::Tensor& uv,
                      const std::optional<torch::Tensor>& gate, int64_t vdim, const torch::Tensor& block_tables,
                      const torch::Tensor& seq_lens, const torch::Tensor& query_start_loc, double scale, int64_t window,
                      int64_t absorbed_max, int64_t max_query_len, int64_t max_seq_len, const std::optional<torch::Tensor>& sink) {
  const char* op = "latent_attention";
  LV_CHECK_DEVICE(q);
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(q));
  TORCH_CHECK(q.dim() == 3 && q.is_contiguous() && q.scalar_type() == cache.scalar_type(), op, ": contiguous q [rows, heads, row]");
  const int64_t rows = q.size(0), heads = q.size(1);
  TORCH_CHECK(uv.is_cuda() && uv.dim() == 3 && uv.is_contiguous() && uv.size(0) == heads && uv.scalar_type() == q.scalar_type(), op,
              ": uv [heads, vpad, cpad]");
  const int64_t cpad = uv.size(2), rpad = q.size(2) - cpad;
  check_latent_rows(cache, cpad, rpad, op);
  check_layout(query_start_loc, seq_lens, op);
  check_tables(block_tables, seq_lens.numel(), op);
  check_rows2d(out, rows, heads * vdim, q.scalar_type(), op, "out");
  if (gate) check_rows2d(*gate, rows, heads, q.scalar_type(), op, "gate");
  if (sink) check_f32(*sink, heads, op, "sink");
  const int ns = (int)seq_lens.numel(), code = dtype_code(q, op), bs = (int)cache.size(1);
  const int64_t need = lvllm_latent_attention_workspace_bytes((int)rows, ns, (int)heads, (int)cpad, (int)rpad, bs, (int)window,
                                                              (int)absorbed_max, (int)max_query_len, (int)max_seq_len, code);
  auto ws = torch::empty({need}, q.options().dtype(at::kByte));
  check(lvllm_latent_attention(out.data_ptr(), out.stride(0), q.data_ptr(), cache.data_ptr(), cache.stride(0), cache.size(0), bs,
                               (int)cpad, (int)rpad, uv.data_ptr(), (int)vdim, (int)uv.size(1),
                               gate ? gate->data_ptr() : nullptr, gate ? gate->stride(0) : 0,
                               sink ? sink->data_ptr<float>() : nullptr, block_tables.data_ptr<int>(),
                               (int)block_tables.size(1), seq_lens.data_ptr<int>(), query_start_loc.data_ptr<int>(), ns,
                               (int)rows, (int)heads, (float)scale, (int)window, (int)absorbed_max, (int)max_query_len,
                               (int)max_seq_len, ws.data_ptr(), need, code, current_stream(q)));
}

torch::Tensor latent_gather(const torch::Tensor& cache, const torch::Tensor& starts, const torch::Tensor& first,
                            const torch::Tensor& seq_lens, const torch::Tensor& block_tables, int64_t n) {
  const char* op = "latent_gather";
  LV_CHECK_DEVICE(cache);
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(cache));
  check_latent_rows(cache, cache.size(2), 0, op);
  const int64_t ns = seq_lens.numel();
  check_i32(seq_lens, ns, op, "seq_lens");
  check_i32(starts, ns + 1, op, "starts");
  check_i32(first, ns, op, "first");
  check_tables(block_tables, ns, op);
  auto out = torch::empty({n, cache.size(2)}, cache.options());
  check(lvllm_latent_gather(out.data_ptr(), cache.data_ptr(), cache.stride(0), cache.size(0), (int)cache.size(1),
                            (int)cache.size(2), starts.data_ptr<int>(), first.data_ptr<int>(), seq_lens.data_ptr<int>(),
                            block_tables.data_ptr<int>(), (int)block_tables.size(1), (int)ns, (int)n, dtype_code(cache, op),
                            current_stream(cache)));
  return out;
}

std::tuple<torch::Tensor, torch::Tensor> latent_expand(const torch::Tensor& kv, const torch::Tensor& rows, int64_t cpad,
                                                       int64_t heads, int64_t dim, int64_t rot_dim, int64_t vdim, int64_t kpad,
                                                       int64_t vpad) {
  const char* op = "latent_expand";
  LV_CHECK_DEVICE(kv);
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(kv));
  const int64_t n = rows.size(0);
  TORCH_CHECK(rows.dim() == 2 && rows.is_contiguous() && rows.scalar_type() == kv.scalar_type() && cpad + rot_dim <= rows.size(1) &&
                  n % 16 == 0,
              op, ": gathered rows [16 n, cpad + rpad]");
  check_rows2d(kv, n, heads * (dim + vdim), rows.scalar_type(), op, "kv");
  auto k = torch::empty({n / 16, heads, kpad / 8, 16, 8}, kv.options());
  auto v = torch::empty({n / 16, heads, vpad, 16}, kv.options());
  check(lvllm_latent_expand(k.data_ptr(), v.data_ptr(), kv.data_ptr(), kv.stride(0), rows.data_ptr(), (int)rows.size(1),
                            (int)cpad, (int)n, (int)heads, (int)dim, (int)rot_dim, (int)vdim, (int)kpad, (int)vpad,
                            dtype_code(kv, op), current_stream(kv)));
  return {k, v};
}

torch::Tensor latent_rotate_query(const torch::Tensor& q, int64_t heads, int64_t dim, int64_t kpad,
                                  const torch::Tensor& positions, const torch::Tensor& turns, double grow) {
  const char* op = "latent_rotate_query";
  LV_CHECK_DEVICE(q);
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(q));
  const int64_t rows = q.size(0);
  TORCH_CHECK(heads > 0 && q.dim() == 2 && q.size(1) % heads == 0 && q.size(1) / heads >= dim, op, ": q [rows, heads * (dim + rot_dim)]");
  check_rows2d(q, rows, q.size(1), q.scalar_type(), op, "q");
  check_rot(positions, turns, rows, op);
  auto out = torch::empty({rows, heads, kpad}, q.options());
  check(lvllm_latent_rotate_query(out.data_ptr(), q.data_ptr(), q.stride(0), (int)heads, (int)dim,
                                  (int)(q.size(1) / heads - dim), (int)kpad, positions.data_ptr<int64_t>(),
                                  turns.data_ptr<double>(), (int)turns.numel() * 2, (float)grow, (int)rows, dtype_code(q, op),
                                  current_stream(q)));
  return out;
}

torch::Tensor embed_scale(torch::Tensor& x, const torch::Tensor& table, const torch::Tensor& ids, double scale) {
  const char* op = "embed_scale";
  check_residual(x, op);
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(x));
  TORCH_CHECK(table.is_cuda() && table.dim() == 2 && table.is_contiguous() && table.size(1) == x.size(1) && ids.is_cuda() &&
                  ids.scalar_type() == at::kLong && ids.is_contiguous() && ids.numel() == x.size(0),
              op, ": table [vocab, width], ids int64 [rows]");
  auto h = torch::empty(x.sizes(), table.options());
  check(lvllm_embed_scale(x.data_ptr<float>(), h.data_ptr(), table.data_ptr(), ids.data_ptr<int64_t>(), (float)scale,
                          (int)x.size(0), (int)table.size(0), (int)x.size(1), dtype_code(table, op), current_stream(x)));
  return h;
}

// y: rows of the compute dtype, fp32 slabs [s, rows, width], or (with slots and weights) the slots of a mixture
torch::Tensor norm_add_mix(const std::optional<torch::Tensor>& x_out, const std::optional<torch::Tensor>& v_out,
                           const torch::Tensor& x, const torch::Tensor& y, const std::optional<torch::Tensor>& slots,
                           const std::optional<torch::Tensor>& slot_weights, const torch::Tensor& gain, double eps,
                           const std::optional<torch::Tensor>& streams, const std::optional<torch::Tensor>& weights,
                           const std::optional<torch::Tensor>& out_gain, at::ScalarType dtype) {
  const char* op = "norm_add_mix";
  check_residual(x, op);
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(x));
  const int64_t rows = x.size(0), width = x.size(1);
  check_f32(gain, 1, op, "gain");
  if (out_gain) check_f32(*out_gain, 1, op, "out_gain");
  for (const auto* t : {&x_out, &v_out})
    if (*t) {
      check_residual(**t, op);
      TORCH_CHECK((*t)->sizes() == x.sizes(), op, ": outputs of the residual's shape");
    }
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
    a = addend_of(y, x, dtype, op);
  }
  int num_streams = 0;
  int64_t stream_stride = 0;
  TORCH_CHECK(!streams || weights, op, ": streams need weights");
  if (weights) {
    num_streams = streams ? (int)streams->size(0) : 0;
    check_f32(*weights, num_streams + 1, op, "weights");
    if (streams) {
      TORCH_CHECK(streams->is_cuda() && streams->dim() == 3 && streams->scalar_type() == at::kFloat && streams->size(1) == rows &&
                      streams->size(2) == width && (rows == 0 || (*streams)[0].is_contiguous()),
                  op, ": streams float32 [n, rows, width], each contiguous");
      stream_stride = streams->stride(0);
    }
  }
  auto h = torch::empty(x.sizes(), x.options().dtype(dtype));
  check(lvllm_norm_add_mix(x_out ? x_out->data_ptr<float>() : nullptr, v_out ? v_out->data_ptr<float>() : nullptr, h.data_ptr(),
                           x.data_ptr<float>(), a.y, a.partials, a.num, slots ? slots->data_ptr<int>() : nullptr,
                           slots ? slot_weights->data_ptr<float>() : nullptr, per_row, total, gain.data_ptr<float>(), (float)eps,
                           streams ? streams->data_ptr<float>() : nullptr, stream_stride, num_streams,
                           weights ? weights->data_ptr<float>() : nullptr, out_gain ? out_gain->data_ptr<float>() : nullptr,
                           (float)eps, (int)rows, (int)width, dtype_code(h, op), current_stream(x)));
  return h;
}

}  // namespace

TORCH_LIBRARY_FRAGMENT(_C_amd, latent) {
  latent.def("latent_cache(Tensor(a!) cache, Tensor kv, Tensor weight, float eps, int cpad, Tensor positions, Tensor turns, "
             "Tensor slot_mapping, float grow=1.) -> ()");
  latent.impl("latent_cache", torch::kCUDA, &latent_cache);
  latent.def("latent_down(Tensor q, Tensor q_weight, int q_pad, Tensor(a!) cache, Tensor kv, Tensor weight, float eps, int cpad, "
             "Tensor positions, Tensor turns, Tensor slot_mapping, float grow=1.) -> Tensor");
  latent.impl("latent_down", torch::kCUDA, &latent_down);
  latent.def("latent_query(Tensor q, Tensor uk_t, int dim, Tensor positions, Tensor turns, Tensor query_start_loc, "
             "int absorbed_max, Tensor(a!) cache, Tensor? kv, Tensor? weight, float eps, Tensor slot_mapping, "
             "float grow=1.) -> Tensor");
  latent.impl("latent_query", torch::kCUDA, &latent_query);
  latent.def("latent_attention(Tensor(a!) out, Tensor q, Tensor cache, Tensor uv, Tensor? gate, int vdim, Tensor block_tables, "
             "Tensor seq_lens, Tensor query_start_loc, float scale, int window, int absorbed_max, int max_query_len, "
             "int max_seq_len, Tensor? sink=None) -> ()");
  latent.impl("latent_attention", torch::kCUDA, &latent_attention);
  latent.def("latent_gather(Tensor cache, Tensor starts, Tensor first, Tensor seq_lens, Tensor block_tables, int n) -> Tensor");
  latent.impl("latent_gather", torch::kCUDA, &latent_gather);
  latent.def("latent_expand(Tensor kv, Tensor rows, int cpad, int heads, int dim, int rot_dim, int vdim, int kpad, int vpad) "
             "-> (Tensor, Tensor)");
  latent.impl("latent_expand", torch::kCUDA, &latent_expand);
  latent.def("latent_rotate_query(Tensor q, int heads, int dim, int kpad, Tensor positions, Tensor turns, "
             "float grow=1.) -> Tensor");
  latent.impl("latent_rotate_query", torch::kCUDA, &latent_rotate_query);
  latent.def("embed_scale(Tensor(a!) x, Tensor table, Tensor ids, float scale) -> Tensor");
  latent.impl("embed_scale", torch::kCUDA, &embed_scale);
  latent.def("norm_add_mix(Tensor(a!)? x_out, Tensor(b!)? v_out, Tensor x, Tensor y, Tensor? slots, Tensor? slot_weights, "
             "Tensor gain, float eps, Tensor? streams, Tensor? weights, Tensor? out_gain, ScalarType dtype) -> Tensor");
  latent.impl("norm_add_mix", torch::kCUDA, &norm_add_mix);
}

PyMODINIT_FUNC PyInit__C_latent(void) {
  static struct PyModuleDef module = {PyModuleDef_HEAD_INIT, "_C_latent", nullptr, 0, nullptr};
  return PyModule_Create(&module);
}
