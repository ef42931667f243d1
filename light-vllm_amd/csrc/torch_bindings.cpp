// torch op registrations: `torch.ops._C.*`, `torch.ops._C_cache_ops.*`,
// `torch.ops._C_cuda_utils.*` with the schemas of the reference
// (csrc/torch_bindings.cpp:18-279), each implemented by unpacking tensors and
// forwarding to the C-ABI of include/lvllm_hip.h on the CURRENT stream of the
// tensor's device (csrc/attention/attention_kernels.cu:736-737 does the same).
//
// Host-only C++ (built with g++): no device code lives here.  The operators every model needs (cache movement, decode
// GEMMs, sampling, step inputs) are registered by torch_bindings_base.cpp.
#include "torch_bindings.h"

namespace {

void paged_attention_v1(torch::Tensor& out, torch::Tensor& query, torch::Tensor& key_cache,
                        torch::Tensor& value_cache, int64_t num_kv_heads, double scale,
                        torch::Tensor& block_tables, torch::Tensor& seq_lens, int64_t block_size,
                        int64_t max_seq_len, const std::optional<torch::Tensor>& alibi_slopes,
                        const std::string& kv_cache_dtype, double k_scale, double v_scale,
                        const int64_t tp_rank, const int64_t blocksparse_local_blocks,
                        const int64_t blocksparse_vert_stride, const int64_t blocksparse_block_size,
                        const int64_t blocksparse_head_sliding_step) {
  LV_CHECK_DEVICE(query);
  TORCH_CHECK(out.is_contiguous(), "out must be contiguous");
  TORCH_CHECK(block_tables.scalar_type() == at::kInt && seq_lens.scalar_type() == at::kInt,
              "block_tables / seq_lens must be int32");
  check_cache_dtype(key_cache, query, kv_dtype_code(kv_cache_dtype), "paged_attention_v1");
  check_cache_dtype(value_cache, query, kv_dtype_code(kv_cache_dtype), "paged_attention_v1");
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(query));
  const float* alibi = alibi_slopes ? alibi_slopes->data_ptr<float>() : nullptr;
  check(lvllm_paged_attention_v1(
      out.data_ptr(), query.data_ptr(), key_cache.data_ptr(), value_cache.data_ptr(),
      (int)query.size(0), (int)query.size(1), (int)query.size(2), (int)num_kv_heads, (float)scale,
      block_tables.data_ptr<int>(), seq_lens.data_ptr<int>(), (int)block_size, (int)max_seq_len,
      (int)block_tables.size(1), alibi, query.stride(0), key_cache.stride(0), key_cache.stride(1),
      dtype_code(query, "paged_attention_v1"), kv_dtype_code(kv_cache_dtype), (float)k_scale,
      (float)v_scale, (int)tp_rank, (int)blocksparse_local_blocks, (int)blocksparse_vert_stride,
      (int)blocksparse_block_size, (int)blocksparse_head_sliding_step, cache_extent_bytes(key_cache, value_cache),
      current_stream(query)));
}

void paged_attention_v2(torch::Tensor& out, torch::Tensor& exp_sums, torch::Tensor& max_logits,
                        torch::Tensor& tmp_out, torch::Tensor& query, torch::Tensor& key_cache,
                        torch::Tensor& value_cache, int64_t num_kv_heads, double scale,
                        torch::Tensor& block_tables, torch::Tensor& seq_lens, int64_t block_size,
                        int64_t max_seq_len, const std::optional<torch::Tensor>& alibi_slopes,
                        const std::string& kv_cache_dtype, double k_scale, double v_scale,
                        const int64_t tp_rank, const int64_t blocksparse_local_blocks,
                        const int64_t blocksparse_vert_stride, const int64_t blocksparse_block_size,
                        const int64_t blocksparse_head_sliding_step) {
  LV_CHECK_DEVICE(query);
  TORCH_CHECK(out.is_contiguous() && tmp_out.is_contiguous() && exp_sums.is_contiguous() &&
                  max_logits.is_contiguous(),
              "out / tmp_out / exp_sums / max_logits must be contiguous");
  TORCH_CHECK(block_tables.scalar_type() == at::kInt && seq_lens.scalar_type() == at::kInt,
              "block_tables / seq_lens must be int32");
  TORCH_CHECK(exp_sums.scalar_type() == at::kFloat && max_logits.scalar_type() == at::kFloat,
              "exp_sums / max_logits must be float32");
  check_cache_dtype(key_cache, query, kv_dtype_code(kv_cache_dtype), "paged_attention_v2");
  check_cache_dtype(value_cache, query, kv_dtype_code(kv_cache_dtype), "paged_attention_v2");
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(query));
  const float* alibi = alibi_slopes ? alibi_slopes->data_ptr<float>() : nullptr;
  check(lvllm_paged_attention_v2(
      out.data_ptr(), exp_sums.data_ptr<float>(), max_logits.data_ptr<float>(), tmp_out.data_ptr(),
      query.data_ptr(), key_cache.data_ptr(), value_cache.data_ptr(), (int)query.size(0),
      (int)query.size(1), (int)query.size(2), (int)num_kv_heads, (float)scale,
      block_tables.data_ptr<int>(), seq_lens.data_ptr<int>(), (int)block_size, (int)max_seq_len,
      (int)block_tables.size(1), (int)exp_sums.size(-1), alibi, query.stride(0),
      key_cache.stride(0), key_cache.stride(1), dtype_code(query, "paged_attention_v2"),
      kv_dtype_code(kv_cache_dtype), (float)k_scale, (float)v_scale, (int)tp_rank,
      (int)blocksparse_local_blocks, (int)blocksparse_vert_stride, (int)blocksparse_block_size,
      (int)blocksparse_head_sliding_step, cache_extent_bytes(key_cache, value_cache), current_stream(query)));
}

void silu_and_mul(torch::Tensor& out, torch::Tensor& input) {
  LV_CHECK_DEVICE(input);
  TORCH_CHECK(input.is_contiguous() && out.is_contiguous(), "silu_and_mul needs contiguous tensors");
  const int64_t d = input.size(-1) / 2;
  const int64_t num_tokens = input.numel() / input.size(-1);
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(input));
  check(lvllm_silu_and_mul(out.data_ptr(), input.data_ptr(), num_tokens, (int)d,
                           dtype_code(input, "silu_and_mul"), current_stream(input)));
}

void rms_norm(torch::Tensor& out, torch::Tensor& input, torch::Tensor& weight, double epsilon) {
  LV_CHECK_DEVICE(input);
  TORCH_CHECK(input.is_contiguous() && out.is_contiguous(), "rms_norm needs contiguous tensors");
  const int hidden = (int)input.size(-1);
  const int num_tokens = (int)(input.numel() / hidden);
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(input));
  check(lvllm_rms_norm(out.data_ptr(), input.data_ptr(), weight.data_ptr(), (float)epsilon,
                       num_tokens, hidden, dtype_code(input, "rms_norm"), current_stream(input)));
}

void fused_add_rms_norm(torch::Tensor& input, torch::Tensor& residual, torch::Tensor& weight,
                        double epsilon) {
  LV_CHECK_DEVICE(input);
  TORCH_CHECK(input.is_contiguous() && residual.is_contiguous(),
              "fused_add_rms_norm needs contiguous tensors");
  const int hidden = (int)input.size(-1);
  const int num_tokens = (int)(input.numel() / hidden);
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(input));
  check(lvllm_fused_add_rms_norm(input.data_ptr(), residual.data_ptr(), weight.data_ptr(),
                                 (float)epsilon, num_tokens, hidden,
                                 dtype_code(input, "fused_add_rms_norm"), current_stream(input)));
}

void rotary_embedding(torch::Tensor& positions, torch::Tensor& query, torch::Tensor& key,
                      int64_t head_size, torch::Tensor& cos_sin_cache, bool is_neox) {
  LV_CHECK_DEVICE(query);
  TORCH_CHECK(positions.scalar_type() == at::kLong, "positions must be int64");
  const int64_t num_tokens = query.numel() / query.size(-1);
  const int rot_dim = (int)cos_sin_cache.size(1);
  const int num_heads = (int)(query.size(-1) / head_size);
  const int num_kv_heads = (int)(key.size(-1) / head_size);
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(query));
  check(lvllm_rotary_embedding(positions.data_ptr<int64_t>(), query.data_ptr(), key.data_ptr(),
                               (int)num_tokens, num_heads, num_kv_heads, (int)head_size, rot_dim,
                               query.stride(-2), key.stride(-2), cos_sin_cache.data_ptr(),
                               is_neox ? 1 : 0, dtype_code(query, "rotary_embedding"),
                               current_stream(query)));
}

void gelu(torch::Tensor& out, const torch::Tensor& x) {
  LV_CHECK_DEVICE(x);
  TORCH_CHECK(x.is_contiguous() && out.is_contiguous() && out.sizes() == x.sizes() && out.scalar_type() == x.scalar_type(),
              "gelu: contiguous out and x of the same shape and type");
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(x));
  check(lvllm_gelu(out.data_ptr(), x.data_ptr(), x.numel(), dtype_code(x, "gelu"), current_stream(x)));
}

void add_layer_norm(torch::Tensor& out, const torch::Tensor& x, const std::optional<torch::Tensor>& y,
                    const torch::Tensor& weight, const torch::Tensor& bias, double epsilon) {
  LV_CHECK_DEVICE(x);
  TORCH_CHECK(x.is_contiguous() && out.is_contiguous() && out.sizes() == x.sizes() && out.scalar_type() == x.scalar_type(),
              "add_layer_norm: contiguous out and x of the same shape and type");
  TORCH_CHECK(!y || (y->is_contiguous() && y->sizes() == x.sizes() && y->scalar_type() == x.scalar_type()),
              "add_layer_norm: y must match x");
  const int hidden = (int)x.size(-1);
  TORCH_CHECK(weight.numel() == hidden && bias.numel() == hidden && weight.is_contiguous() && bias.is_contiguous() &&
                  weight.scalar_type() == x.scalar_type() && bias.scalar_type() == x.scalar_type(),
              "add_layer_norm: weight and bias of [hidden] in x's type");
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(x));
  check(lvllm_add_layer_norm(out.data_ptr(), x.data_ptr(), y ? y->data_ptr() : nullptr, weight.data_ptr(),
                             bias.data_ptr(), (float)epsilon, (int)(x.numel() / hidden), hidden,
                             dtype_code(x, "add_layer_norm"), current_stream(x)));
}

void fused_add_rms_norm_splitk_scaled(torch::Tensor& out, torch::Tensor& residual, const torch::Tensor& partials,
                                      const torch::Tensor& weight, double epsilon,
                                      const c10::optional<torch::Tensor>& x_scale,
                                      const c10::optional<torch::Tensor>& w_scale) {
  TORCH_CHECK(partials.dim() == 3 && partials.scalar_type() == at::kFloat && partials.is_contiguous());
  TORCH_CHECK(out.is_contiguous() && residual.is_contiguous() && out.sizes() == residual.sizes());
  TORCH_CHECK(x_scale.has_value() == w_scale.has_value(), "x_scale and w_scale: both or none");
  if (x_scale.has_value())
    TORCH_CHECK(x_scale->scalar_type() == at::kFloat && w_scale->scalar_type() == at::kFloat && x_scale->is_cuda() &&
                w_scale->is_cuda() && x_scale->numel() == 1 && w_scale->numel() == 1, "scales: one float each, on the GPU");
  const int hidden = (int)out.size(-1);
  const int num_tokens = (int)(out.numel() / hidden);
  TORCH_CHECK(partials.size(1) == num_tokens && partials.size(2) == hidden);
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(out));
  check(lvllm_fused_add_rms_norm_splitk_scaled(
      out.data_ptr(), residual.data_ptr(), partials.data_ptr<float>(), (int)partials.size(0), weight.data_ptr(),
      (float)epsilon, num_tokens, hidden, dtype_code(out, "fused_add_rms_norm_splitk"),
      x_scale.has_value() ? x_scale->data_ptr<float>() : nullptr,
      w_scale.has_value() ? w_scale->data_ptr<float>() : nullptr, current_stream(out)));
}

void fused_add_rms_norm_splitk(torch::Tensor& out, torch::Tensor& residual, const torch::Tensor& partials,
                               const torch::Tensor& weight, double epsilon) {
  fused_add_rms_norm_splitk_scaled(out, residual, partials, weight, epsilon, c10::nullopt, c10::nullopt);
}

// returns false when the arguments are outside the fused kernel's envelope (nothing was done)
bool rotary_embedding_and_cache(torch::Tensor& positions, torch::Tensor& query, torch::Tensor& key,
                                const torch::Tensor& value, int64_t head_size, torch::Tensor& cos_sin_cache,
                                bool is_neox, torch::Tensor& key_cache, torch::Tensor& value_cache,
                                const torch::Tensor& slot_mapping, const std::string& kv_cache_dtype,
                                double k_scale, double v_scale) {
  LV_CHECK_DEVICE(query);
  TORCH_CHECK(positions.scalar_type() == at::kLong && slot_mapping.scalar_type() == at::kLong);
  const int kv_code = kv_dtype_code(kv_cache_dtype);
  check_cache_dtype(key_cache, query, kv_code, "rotary_embedding_and_cache");
  check_cache_dtype(value_cache, query, kv_code, "rotary_embedding_and_cache");
  const int64_t num_tokens = query.numel() / query.size(-1);
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(query));
  TORCH_CHECK(blocks_are_dense(key_cache) && blocks_are_dense(value_cache) &&
                  key_cache.stride(0) == value_cache.stride(0),
              "key_cache / value_cache: dense blocks, the same block stride");
  const int rc = lvllm_rotary_embedding_and_cache_strided(
      positions.data_ptr<int64_t>(), query.data_ptr(), key.data_ptr(), value.data_ptr(), (int)num_tokens,
      (int)(query.size(-1) / head_size), (int)(key.size(-1) / head_size), (int)head_size,
      (int)cos_sin_cache.size(1), query.stride(-2), key.stride(-2), value.stride(-2), cos_sin_cache.data_ptr(),
      is_neox ? 1 : 0, key_cache.data_ptr(), value_cache.data_ptr(), slot_mapping.data_ptr<int64_t>(),
      (int)value_cache.size(3), dtype_code(query, "rotary_embedding_and_cache"), kv_code, (float)k_scale,
      (float)v_scale, cache_extent_bytes(key_cache, value_cache), key_cache.stride(0), current_stream(query));
  if (rc == 3) return false;
  check(rc);
  return true;
}

// the QKV projection's split-K reduce + rope + cache write in one launch (include/lvllm_hip.h); false = outside the
// fused kernel's envelope (nothing was done)
bool rotary_embedding_and_cache_splitk(torch::Tensor& positions, torch::Tensor& qkv, const torch::Tensor& partials,
                                       const std::optional<torch::Tensor>& bias, int64_t num_heads, int64_t num_kv_heads,
                                       int64_t head_size, torch::Tensor& cos_sin_cache, bool is_neox,
                                       torch::Tensor& key_cache, torch::Tensor& value_cache,
                                       const torch::Tensor& slot_mapping, const std::string& kv_cache_dtype,
                                       double k_scale, double v_scale) {
  LV_CHECK_DEVICE(qkv);
  TORCH_CHECK(positions.scalar_type() == at::kLong && slot_mapping.scalar_type() == at::kLong);
  const int64_t row = (num_heads + 2 * num_kv_heads) * head_size;
  TORCH_CHECK(qkv.dim() == 2 && qkv.is_contiguous() && qkv.size(1) == row, "qkv: contiguous [tokens, (H + 2 KVH) * D]");
  TORCH_CHECK(partials.scalar_type() == at::kFloat && partials.is_contiguous() && partials.dim() == 3 &&
                  partials.size(1) == qkv.size(0) && partials.size(2) == row && partials.device() == qkv.device(),
              "partials: contiguous fp32 [slabs, tokens, (H + 2 KVH) * D] on qkv's device");
  TORCH_CHECK(!bias.has_value() || (bias->numel() == row && bias->scalar_type() == qkv.scalar_type() && bias->is_contiguous()),
              "bias: [(H + 2 KVH) * D] of qkv's type");
  const int kv_code = kv_dtype_code(kv_cache_dtype);
  check_cache_dtype(key_cache, qkv, kv_code, "rotary_embedding_and_cache_splitk");
  check_cache_dtype(value_cache, qkv, kv_code, "rotary_embedding_and_cache_splitk");
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(qkv));
  TORCH_CHECK(blocks_are_dense(key_cache) && blocks_are_dense(value_cache) &&
                  key_cache.stride(0) == value_cache.stride(0),
              "key_cache / value_cache: dense blocks, the same block stride");
  const int rc = lvllm_rotary_embedding_and_cache_splitk(
      positions.data_ptr<int64_t>(), qkv.data_ptr(), partials.data_ptr<float>(), (int)partials.size(0),
      bias.has_value() ? bias->data_ptr() : nullptr, (int)qkv.size(0), (int)num_heads, (int)num_kv_heads, (int)head_size,
      (int)cos_sin_cache.size(1), cos_sin_cache.data_ptr(), is_neox ? 1 : 0, key_cache.data_ptr(), value_cache.data_ptr(),
      slot_mapping.data_ptr<int64_t>(), (int)value_cache.size(3), dtype_code(qkv, "rotary_embedding_and_cache_splitk"),
      kv_code, (float)k_scale, (float)v_scale, cache_extent_bytes(key_cache, value_cache), key_cache.stride(0),
      current_stream(qkv));
  if (rc == 3) return false;
  check(rc);
  return true;
}

// returns false when the arguments are outside the fused kernel's envelope (nothing was done)
bool rope_cache_paged_attention(torch::Tensor& out, torch::Tensor& exp_sums, torch::Tensor& max_logits,
                                torch::Tensor& tmp_out, const torch::Tensor& positions, const torch::Tensor& query,
                                const torch::Tensor& key, const torch::Tensor& value, int64_t head_size,
                                const torch::Tensor& cos_sin_cache, bool is_neox, torch::Tensor& key_cache,
                                torch::Tensor& value_cache, const torch::Tensor& slot_mapping, int64_t num_kv_heads,
                                double scale, const torch::Tensor& block_tables, const torch::Tensor& seq_lens,
                                int64_t block_size, int64_t max_seq_len, const std::string& kv_cache_dtype,
                                double k_scale, double v_scale, const c10::optional<torch::Tensor>& out_fp8,
                                const c10::optional<torch::Tensor>& out_fp8_scale) {
  LV_CHECK_DEVICE(query);
  TORCH_CHECK(positions.scalar_type() == at::kLong && slot_mapping.scalar_type() == at::kLong);
  TORCH_CHECK(out_fp8.has_value() == out_fp8_scale.has_value(), "out_fp8 and out_fp8_scale: both or none");
  if (out_fp8.has_value())
    TORCH_CHECK(out_fp8->is_cuda() && out_fp8->element_size() == 1 && out_fp8->is_contiguous() &&
                out_fp8->numel() == out.numel() && out_fp8_scale->is_cuda() && out_fp8_scale->scalar_type() == at::kFloat &&
                out_fp8_scale->numel() == 1, "out_fp8: bytes of out's shape; out_fp8_scale: one float on the device");
  TORCH_CHECK(query.dim() == 2 && key.dim() == 2 && value.dim() == 2, "query / key / value must be [tokens, heads * head_size]");
  TORCH_CHECK(block_tables.scalar_type() == at::kInt && seq_lens.scalar_type() == at::kInt,
              "block_tables / seq_lens must be int32");
  TORCH_CHECK(out.is_contiguous() && tmp_out.is_contiguous() && exp_sums.is_contiguous() && max_logits.is_contiguous());
  const int kv_code = kv_dtype_code(kv_cache_dtype);
  check_cache_dtype(key_cache, query, kv_code, "rope_cache_paged_attention");
  check_cache_dtype(value_cache, query, kv_code, "rope_cache_paged_attention");
  const int64_t num_seqs = query.numel() / query.size(-1);
  const int64_t num_heads = query.size(-1) / head_size;
  TORCH_CHECK(key.size(-1) == num_kv_heads * head_size && value.size(-1) == num_kv_heads * head_size);
  TORCH_CHECK(out.numel() == num_seqs * num_heads * head_size);
  TORCH_CHECK(positions.numel() >= num_seqs && slot_mapping.numel() >= num_seqs && seq_lens.numel() >= num_seqs &&
              block_tables.size(0) >= num_seqs);
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(query));
  const int rc = out_fp8.has_value() ? lvllm_rope_cache_paged_attention_q(
      out.data_ptr(), out_fp8->data_ptr(), out_fp8_scale->data_ptr<float>(), exp_sums.data_ptr<float>(),
      max_logits.data_ptr<float>(), tmp_out.data_ptr(), query.data_ptr(),
      key.data_ptr(), value.data_ptr(), key_cache.data_ptr(), value_cache.data_ptr(), (int)num_seqs, (int)num_heads,
      (int)head_size, (int)num_kv_heads, (float)scale, block_tables.data_ptr<int32_t>(), seq_lens.data_ptr<int32_t>(),
      positions.data_ptr<int64_t>(), slot_mapping.data_ptr<int64_t>(), cos_sin_cache.data_ptr(),
      (int)cos_sin_cache.size(1), is_neox ? 1 : 0, (int)block_size, (int)max_seq_len, (int)block_tables.size(1),
      (int)exp_sums.size(-1), query.stride(-2), key.stride(-2), value.stride(-2), key_cache.stride(0),
      key_cache.stride(1), dtype_code(query, "rope_cache_paged_attention"), kv_code, (float)k_scale, (float)v_scale,
      cache_extent_bytes(key_cache, value_cache), current_stream(query))
                                     : lvllm_rope_cache_paged_attention(
      out.data_ptr(), exp_sums.data_ptr<float>(), max_logits.data_ptr<float>(), tmp_out.data_ptr(), query.data_ptr(),
      key.data_ptr(), value.data_ptr(), key_cache.data_ptr(), value_cache.data_ptr(), (int)num_seqs, (int)num_heads,
      (int)head_size, (int)num_kv_heads, (float)scale, block_tables.data_ptr<int32_t>(), seq_lens.data_ptr<int32_t>(),
      positions.data_ptr<int64_t>(), slot_mapping.data_ptr<int64_t>(), cos_sin_cache.data_ptr(),
      (int)cos_sin_cache.size(1), is_neox ? 1 : 0, (int)block_size, (int)max_seq_len, (int)block_tables.size(1),
      (int)exp_sums.size(-1), query.stride(-2), key.stride(-2), value.stride(-2), key_cache.stride(0),
      key_cache.stride(1), dtype_code(query, "rope_cache_paged_attention"), kv_code, (float)k_scale, (float)v_scale,
      cache_extent_bytes(key_cache, value_cache), current_stream(query));
  if (rc == 3) return false;
  check(rc);
  return true;
}

// paged_attention_v2 with an fp8 twin of its result (lvllm_paged_attention_v2_q); false = the launch would be cut into
// shares (nothing was done: call paged_attention_v2)
bool paged_attention_v2_q(torch::Tensor& out, torch::Tensor& out_fp8, const torch::Tensor& out_fp8_scale,
                          torch::Tensor& exp_sums, torch::Tensor& max_logits, torch::Tensor& tmp_out,
                          const torch::Tensor& query, const torch::Tensor& key_cache, const torch::Tensor& value_cache,
                          int64_t num_kv_heads, double scale, const torch::Tensor& block_tables,
                          const torch::Tensor& seq_lens, int64_t block_size, int64_t max_seq_len,
                          const std::string& kv_cache_dtype, double k_scale, double v_scale) {
  LV_CHECK_DEVICE(query);
  TORCH_CHECK(query.dim() == 3 && out.is_contiguous() && out.sizes() == query.sizes(), "query / out: [seqs, heads, head_size]");
  TORCH_CHECK(out_fp8.is_cuda() && out_fp8.element_size() == 1 && out_fp8.is_contiguous() && out_fp8.numel() == out.numel() &&
              out_fp8_scale.is_cuda() && out_fp8_scale.scalar_type() == at::kFloat && out_fp8_scale.numel() == 1,
              "out_fp8: bytes of out's shape; out_fp8_scale: one float on the device");
  TORCH_CHECK(block_tables.scalar_type() == at::kInt && seq_lens.scalar_type() == at::kInt, "block_tables / seq_lens must be int32");
  const int kv_code = kv_dtype_code(kv_cache_dtype);
  check_cache_dtype(key_cache, query, kv_code, "paged_attention_v2_q");
  check_cache_dtype(value_cache, query, kv_code, "paged_attention_v2_q");
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(query));
  const int rc = lvllm_paged_attention_v2_q(
      out.data_ptr(), out_fp8.data_ptr(), out_fp8_scale.data_ptr<float>(), exp_sums.data_ptr<float>(),
      max_logits.data_ptr<float>(), tmp_out.data_ptr(), query.data_ptr(), key_cache.data_ptr(), value_cache.data_ptr(),
      (int)query.size(0), (int)query.size(1), (int)query.size(2), (int)num_kv_heads, (float)scale,
      block_tables.data_ptr<int32_t>(), seq_lens.data_ptr<int32_t>(), (int)block_size, (int)max_seq_len,
      (int)block_tables.size(1), (int)exp_sums.size(-1), query.stride(0), key_cache.stride(0), key_cache.stride(1),
      dtype_code(query, "paged_attention_v2_q"), kv_code, (float)k_scale, (float)v_scale,
      cache_extent_bytes(key_cache, value_cache), current_stream(query));
  if (rc == 3) return false;
  check(rc);
  return true;
}

void paged_prefill_attention(torch::Tensor& out, const torch::Tensor& query, const torch::Tensor& key_cache,
                             const torch::Tensor& value_cache, int64_t num_kv_heads, double scale,
                             const torch::Tensor& block_tables, const torch::Tensor& seq_lens,
                             const torch::Tensor& query_start_loc, int64_t max_query_len, int64_t block_size,
                             const c10::optional<torch::Tensor>& alibi_slopes, int64_t sliding_window,
                             double softcap, const std::string& kv_cache_dtype, bool causal, double k_scale,
                             double v_scale, int64_t max_seq_len) {
  LV_CHECK_DEVICE(query);
  LV_CHECK_DEVICE(out);
  check_cache_dtype(key_cache, query, kv_dtype_code(kv_cache_dtype), "paged_prefill_attention");
  check_cache_dtype(value_cache, query, kv_dtype_code(kv_cache_dtype), "paged_prefill_attention");
  TORCH_CHECK(query.dim() == 3 && out.dim() == 3, "paged_prefill_attention: query/out must be [T, H, D]");
  TORCH_CHECK(query.stride(2) == 1 && query.stride(1) == query.size(2) && out.stride(2) == 1 &&
                  out.stride(1) == out.size(2),
              "paged_prefill_attention: heads of a token must be contiguous");
  TORCH_CHECK(block_tables.scalar_type() == at::kInt && seq_lens.scalar_type() == at::kInt &&
                  query_start_loc.scalar_type() == at::kInt,
              "paged_prefill_attention: block_tables / seq_lens / query_start_loc must be int32");
  TORCH_CHECK(block_tables.dim() == 2 && block_tables.is_contiguous());
  const int64_t num_seqs = seq_lens.numel();
  TORCH_CHECK(query_start_loc.numel() == num_seqs + 1 && block_tables.size(0) >= num_seqs);
  TORCH_CHECK(value_cache.size(3) == block_size, "paged_prefill_attention: block_size does not match the cache");
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(query));
  const float* alibi = alibi_slopes.has_value() ? alibi_slopes->data_ptr<float>() : nullptr;
  // short chunks with a known bound on seq_lens: scratch for a partitioned key walk (0 bytes: single pass)
  torch::Tensor workspace;
  const int64_t ws_bytes =
      max_seq_len > 0 ? lvllm_paged_prefill_workspace_bytes((int)num_seqs, (int)query.size(0), (int)max_query_len,
                                                            (int)query.size(1), (int)num_kv_heads, (int)query.size(2),
                                                            (int)max_seq_len)
                      : 0;
  if (ws_bytes > 0) workspace = torch::empty({ws_bytes}, query.options().dtype(torch::kUInt8));
  check(lvllm_paged_prefill_attention_ws(
      out.data_ptr(), query.data_ptr(), key_cache.data_ptr(), value_cache.data_ptr(), (int)num_seqs,
      (int)query.size(1), (int)query.size(2), (int)num_kv_heads, (float)scale, block_tables.data_ptr<int32_t>(),
      seq_lens.data_ptr<int32_t>(), query_start_loc.data_ptr<int32_t>(), (int)max_query_len, (int)block_size,
      (int)block_tables.size(1), alibi, causal ? 1 : 0, (int)sliding_window, (float)softcap, query.stride(0),
      out.stride(0),
      key_cache.stride(0), key_cache.stride(1), dtype_code(query, "paged_prefill_attention"),
      kv_dtype_code(kv_cache_dtype), (float)k_scale, (float)v_scale, cache_extent_bytes(key_cache, value_cache),
      (int)query.size(0), (int)max_seq_len, ws_bytes > 0 ? workspace.data_ptr() : nullptr, ws_bytes,
      current_stream(query)));
}

int64_t paged_prefill_workspace_bytes(int64_t num_seqs, int64_t num_tokens, int64_t max_query_len, int64_t num_heads,
                                      int64_t num_kv_heads, int64_t head_size, int64_t max_seq_len) {
  return lvllm_paged_prefill_workspace_bytes((int)num_seqs, (int)num_tokens, (int)max_query_len, (int)num_heads,
                                             (int)num_kv_heads, (int)head_size, (int)max_seq_len);
}

int64_t varlen_attention_workspace_bytes(int64_t num_tokens, int64_t num_seqs, int64_t max_seq_len,
                                         int64_t num_kv_heads, int64_t head_size) {
  return lvllm_varlen_attention_workspace_bytes((int)num_tokens, (int)num_seqs, (int)max_seq_len,
                                                (int)num_kv_heads, (int)head_size);
}

void varlen_attention(torch::Tensor& out, const torch::Tensor& query, const torch::Tensor& key,
                      const torch::Tensor& value, const torch::Tensor& cu_seqlens, int64_t max_seq_len,
                      double scale, bool causal, const c10::optional<torch::Tensor>& alibi_slopes,
                      int64_t sliding_window, double softcap, torch::Tensor& workspace) {
  LV_CHECK_DEVICE(query);
  LV_CHECK_DEVICE(key);
  LV_CHECK_DEVICE(value);
  LV_CHECK_DEVICE(out);
  LV_CHECK_DEVICE(workspace);
  TORCH_CHECK(query.dim() == 3 && key.dim() == 3 && value.dim() == 3 && out.dim() == 3,
              "varlen_attention: query/key/value/out must be [T, heads, D]");
  for (const torch::Tensor* t : {&query, &key, &value, (const torch::Tensor*)&out})
    TORCH_CHECK(t->stride(2) == 1 && t->stride(1) == t->size(2), "varlen_attention: heads of a token must be contiguous");
  TORCH_CHECK(cu_seqlens.scalar_type() == at::kInt && cu_seqlens.is_cuda() && cu_seqlens.is_contiguous(),
              "varlen_attention: cu_seqlens must be a contiguous int32 device tensor");
  TORCH_CHECK(key.scalar_type() == query.scalar_type() && value.scalar_type() == query.scalar_type());
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(query));
  const float* alibi = alibi_slopes.has_value() ? alibi_slopes->data_ptr<float>() : nullptr;
  check(lvllm_varlen_attention(out.data_ptr(), query.data_ptr(), key.data_ptr(), value.data_ptr(),
                               cu_seqlens.data_ptr<int32_t>(), (int)query.size(0), (int)cu_seqlens.numel() - 1,
                               (int)max_seq_len, (int)query.size(1), (int)key.size(1), (int)query.size(2),
                               (float)scale, causal ? 1 : 0, alibi, (int)sliding_window, (float)softcap,
                               query.stride(0), key.stride(0), value.stride(0), out.stride(0),
                               dtype_code(query, "varlen_attention"), workspace.data_ptr(),
                               (int64_t)workspace.nbytes(), current_stream(query)));
}

// fp8 activation quantisation, csrc/quantization/fp8/common.cu:226-292
void check_fp8_out(const torch::Tensor& out, const torch::Tensor& input, const char* op) {
  LV_CHECK_DEVICE(input);
  TORCH_CHECK(out.element_size() == 1, op, ": out must be a float8_e4m3fn (one-byte) tensor");
  TORCH_CHECK(input.is_contiguous() && out.is_contiguous(), op, ": input / out must be contiguous");
}

void static_scaled_fp8_quant(torch::Tensor& out, torch::Tensor const& input, torch::Tensor const& scale) {
  check_fp8_out(out, input, "static_scaled_fp8_quant");
  TORCH_CHECK(scale.scalar_type() == at::kFloat && scale.is_cuda());
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(input));
  check(lvllm_static_scaled_fp8_quant(out.data_ptr(), input.data_ptr(), scale.data_ptr<float>(), input.numel(),
                                      dtype_code(input, "static_scaled_fp8_quant"), current_stream(input)));
}

void dynamic_scaled_fp8_quant(torch::Tensor& out, torch::Tensor const& input, torch::Tensor& scale) {
  check_fp8_out(out, input, "dynamic_scaled_fp8_quant");
  TORCH_CHECK(scale.scalar_type() == at::kFloat && scale.is_cuda());
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(input));
  check(lvllm_dynamic_scaled_fp8_quant(out.data_ptr(), input.data_ptr(), scale.data_ptr<float>(), input.numel(),
                                       dtype_code(input, "dynamic_scaled_fp8_quant"), current_stream(input)));
}

void dynamic_per_token_scaled_fp8_quant(torch::Tensor& out, torch::Tensor const& input, torch::Tensor& scales,
                                        std::optional<at::Tensor> const& scale_ub) {
  check_fp8_out(out, input, "dynamic_per_token_scaled_fp8_quant");
  TORCH_CHECK(scales.scalar_type() == at::kFloat && scales.is_cuda() && scales.is_contiguous());
  const int64_t hidden = input.size(-1);
  const int64_t tokens = input.numel() / hidden;
  TORCH_CHECK(scales.numel() >= tokens);
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(input));
  check(lvllm_dynamic_per_token_scaled_fp8_quant(
      out.data_ptr(), scales.data_ptr<float>(), input.data_ptr(),
      scale_ub.has_value() ? scale_ub->data_ptr<float>() : nullptr, (int)tokens, (int)hidden,
      dtype_code(input, "dynamic_per_token_scaled_fp8_quant"), current_stream(input)));
}

// x_fp8 [T, hidden] uint8 = quant(rms_norm(input) * weight)
torch::Tensor rms_norm_fp8(const torch::Tensor& input, const torch::Tensor& weight, double epsilon,
                           const torch::Tensor& q_scale) {
  LV_CHECK_DEVICE(input);
  check_q_scale(q_scale, "rms_norm_fp8");
  TORCH_CHECK(input.dim() == 2 && input.is_contiguous() && weight.is_contiguous() && weight.numel() == input.size(1));
  auto out8 = torch::empty(input.sizes(), input.options().dtype(torch::kUInt8));
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(input));
  check(lvllm_rms_norm_quant(nullptr, out8.data_ptr(), q_scale.data_ptr<float>(), input.data_ptr(), weight.data_ptr(),
                             (float)epsilon, (int)input.size(0), (int)input.size(1), dtype_code(input, "rms_norm_fp8"),
                             current_stream(input)));
  return out8;
}

// residual <- input + residual; x_fp8 = quant(norm(residual) * weight); `input` is only read
torch::Tensor fused_add_rms_norm_fp8(const torch::Tensor& input, torch::Tensor& residual, const torch::Tensor& weight,
                                     double epsilon, const torch::Tensor& q_scale) {
  LV_CHECK_DEVICE(input);
  check_q_scale(q_scale, "fused_add_rms_norm_fp8");
  TORCH_CHECK(input.dim() == 2 && input.is_contiguous() && residual.is_contiguous() && input.sizes() == residual.sizes() &&
              input.scalar_type() == residual.scalar_type() && weight.is_contiguous() && weight.numel() == input.size(1));
  auto out8 = torch::empty(input.sizes(), input.options().dtype(torch::kUInt8));
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(input));
  check(lvllm_fused_add_rms_norm_quant(const_cast<void*>(input.data_ptr()), residual.data_ptr(), weight.data_ptr(),
                                       (float)epsilon, (int)input.size(0), (int)input.size(1),
                                       dtype_code(input, "fused_add_rms_norm_fp8"), out8.data_ptr(),
                                       q_scale.data_ptr<float>(), 0, current_stream(input)));
  return out8;
}

// the same behind a projection that left its fp32 split-K partials [S, T, hidden] (x_scale / w_scale: a W8A8 one)
torch::Tensor fused_add_rms_norm_splitk_fp8(torch::Tensor& residual, const torch::Tensor& partials,
                                            const torch::Tensor& weight, double epsilon,
                                            const c10::optional<torch::Tensor>& x_scale,
                                            const c10::optional<torch::Tensor>& w_scale, const torch::Tensor& q_scale) {
  LV_CHECK_DEVICE(residual);
  check_q_scale(q_scale, "fused_add_rms_norm_splitk_fp8");
  TORCH_CHECK(partials.dim() == 3 && partials.scalar_type() == at::kFloat && partials.is_contiguous());
  TORCH_CHECK(residual.dim() == 2 && residual.is_contiguous() && partials.size(1) == residual.size(0) &&
              partials.size(2) == residual.size(1));
  TORCH_CHECK(x_scale.has_value() == w_scale.has_value(), "x_scale and w_scale: both or none");
  if (x_scale.has_value()) {
    check_q_scale(*x_scale, "fused_add_rms_norm_splitk_fp8");
    check_q_scale(*w_scale, "fused_add_rms_norm_splitk_fp8");
  }
  auto out8 = torch::empty(residual.sizes(), residual.options().dtype(torch::kUInt8));
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(residual));
  check(lvllm_fused_add_rms_norm_splitk_quant(
      nullptr, residual.data_ptr(), partials.data_ptr<float>(), (int)partials.size(0), weight.data_ptr(), (float)epsilon,
      (int)residual.size(0), (int)residual.size(1), dtype_code(residual, "fused_add_rms_norm_splitk_fp8"),
      x_scale.has_value() ? x_scale->data_ptr<float>() : nullptr, w_scale.has_value() ? w_scale->data_ptr<float>() : nullptr,
      out8.data_ptr(), q_scale.data_ptr<float>(), current_stream(residual)));
  return out8;
}
}  // namespace

// Same namespaces, names and schema strings as csrc/torch_bindings.cpp:18-279
// for the operators on the paged-attention decode path.
TORCH_LIBRARY_FRAGMENT(_C, ops) {
  ops.def(
      "paged_attention_v1("
      "    Tensor! out, Tensor query, Tensor key_cache,"
      "    Tensor value_cache, int num_kv_heads, float scale,"
      "    Tensor block_tables, Tensor seq_lens, int block_size,"
      "    int max_seq_len, Tensor? alibi_slopes,"
      "    str kv_cache_dtype, float k_scale, float v_scale,"
      "    int tp_rank, int blocksparse_local_blocks,"
      "    int blocksparse_vert_stride, int blocksparse_block_size,"
      "    int blocksparse_head_sliding_step) -> ()");
  ops.impl("paged_attention_v1", torch::kCUDA, &paged_attention_v1);

  ops.def(
      "paged_attention_v2("
      "    Tensor! out, Tensor exp_sums, Tensor max_logits,"
      "    Tensor tmp_out, Tensor query, Tensor key_cache,"
      "    Tensor value_cache, int num_kv_heads, float scale,"
      "    Tensor block_tables, Tensor seq_lens, int block_size,"
      "    int max_seq_len, Tensor? alibi_slopes,"
      "    str kv_cache_dtype, float k_scale, float v_scale,"
      "    int tp_rank, int blocksparse_local_blocks,"
      "    int blocksparse_vert_stride, int blocksparse_block_size,"
      "    int blocksparse_head_sliding_step) -> ()");
  ops.impl("paged_attention_v2", torch::kCUDA, &paged_attention_v2);

  // fp8 activation quantisation (torch_bindings.cpp:185-202 of the reference)
  ops.def("static_scaled_fp8_quant(Tensor! out, Tensor input, Tensor scale) -> ()");
  ops.impl("static_scaled_fp8_quant", torch::kCUDA, &static_scaled_fp8_quant);
  ops.def("dynamic_scaled_fp8_quant(Tensor! out, Tensor input, Tensor! scale) -> ()");
  ops.impl("dynamic_scaled_fp8_quant", torch::kCUDA, &dynamic_scaled_fp8_quant);
  ops.def("dynamic_per_token_scaled_fp8_quant(Tensor! out, Tensor input, Tensor! scale, Tensor? scale_ub) -> ()");
  ops.impl("dynamic_per_token_scaled_fp8_quant", torch::kCUDA, &dynamic_per_token_scaled_fp8_quant);

  ops.def("silu_and_mul(Tensor! out, Tensor input) -> ()");
  ops.impl("silu_and_mul", torch::kCUDA, &silu_and_mul);

  ops.def("rms_norm(Tensor! out, Tensor input, Tensor weight, float epsilon) -> ()");
  ops.impl("rms_norm", torch::kCUDA, &rms_norm);

  ops.def(
      "fused_add_rms_norm(Tensor! input, Tensor! residual, Tensor weight, "
      "float epsilon) -> ()");
  ops.impl("fused_add_rms_norm", torch::kCUDA, &fused_add_rms_norm);

  ops.def(
      "rotary_embedding(Tensor positions, Tensor! query,"
      "                 Tensor! key, int head_size,"
      "                 Tensor cos_sin_cache, bool is_neox) -> ()");
  ops.impl("rotary_embedding", torch::kCUDA, &rotary_embedding);
}


// operators this build adds beyond the reference's list
TORCH_LIBRARY_FRAGMENT(_C_amd, amd) {
  amd.def("gelu(Tensor! out, Tensor x) -> ()");
  amd.impl("gelu", torch::kCUDA, &gelu);
  amd.def("add_layer_norm(Tensor! out, Tensor x, Tensor? y, Tensor weight, Tensor bias, float epsilon) -> ()");
  amd.impl("add_layer_norm", torch::kCUDA, &add_layer_norm);
  amd.def("fused_add_rms_norm_splitk(Tensor! out, Tensor! residual, Tensor partials, Tensor weight, "
          "float epsilon) -> ()");
  amd.impl("fused_add_rms_norm_splitk", torch::kCUDA, &fused_add_rms_norm_splitk);
  amd.def("rotary_embedding_and_cache(Tensor positions, Tensor! query, Tensor! key, Tensor value, "
          "int head_size, Tensor cos_sin_cache, bool is_neox, Tensor! key_cache, Tensor! value_cache, "
          "Tensor slot_mapping, str kv_cache_dtype=\"auto\", float k_scale=1.0, float v_scale=1.0) -> bool");
  amd.impl("rotary_embedding_and_cache", torch::kCUDA, &rotary_embedding_and_cache);
  amd.def("rotary_embedding_and_cache_splitk(Tensor positions, Tensor! qkv, Tensor partials, Tensor? bias, "
          "int num_heads, int num_kv_heads, int head_size, Tensor cos_sin_cache, bool is_neox, Tensor! key_cache, "
          "Tensor! value_cache, Tensor slot_mapping, str kv_cache_dtype=\"auto\", float k_scale=1.0, "
          "float v_scale=1.0) -> bool");
  amd.impl("rotary_embedding_and_cache_splitk", torch::kCUDA, &rotary_embedding_and_cache_splitk);
  amd.def("paged_prefill_attention(Tensor! out, Tensor query, Tensor key_cache, Tensor value_cache, "
          "int num_kv_heads, float scale, Tensor block_tables, Tensor seq_lens, Tensor query_start_loc, "
          "int max_query_len, int block_size, Tensor? alibi_slopes, int sliding_window, float softcap, "
          "str kv_cache_dtype, bool causal=True, float k_scale=1.0, float v_scale=1.0, int max_seq_len=0) -> ()");
  amd.impl("paged_prefill_attention", torch::kCUDA, &paged_prefill_attention);
  amd.def("rope_cache_paged_attention(Tensor! out, Tensor! exp_sums, Tensor! max_logits, Tensor! tmp_out, "
          "Tensor positions, Tensor query, Tensor key, Tensor value, int head_size, Tensor cos_sin_cache, "
          "bool is_neox, Tensor! key_cache, Tensor! value_cache, Tensor slot_mapping, int num_kv_heads, "
          "float scale, Tensor block_tables, Tensor seq_lens, int block_size, int max_seq_len, "
          "str kv_cache_dtype, float k_scale=1.0, float v_scale=1.0, Tensor(a!)? out_fp8=None, "
          "Tensor? out_fp8_scale=None) -> bool");
  amd.impl("rope_cache_paged_attention", torch::kCUDA, &rope_cache_paged_attention);
  amd.def("paged_attention_v2_q(Tensor! out, Tensor! out_fp8, Tensor out_fp8_scale, Tensor! exp_sums, Tensor! max_logits, "
          "Tensor! tmp_out, Tensor query, Tensor key_cache, Tensor value_cache, int num_kv_heads, float scale, "
          "Tensor block_tables, Tensor seq_lens, int block_size, int max_seq_len, str kv_cache_dtype, "
          "float k_scale=1.0, float v_scale=1.0) -> bool");
  amd.impl("paged_attention_v2_q", torch::kCUDA, &paged_attention_v2_q);
  amd.def("fused_add_rms_norm_splitk_scaled(Tensor! out, Tensor! residual, Tensor partials, Tensor weight, "
          "float epsilon, Tensor? x_scale, Tensor? w_scale) -> ()");
  amd.impl("fused_add_rms_norm_splitk_scaled", torch::kCUDA, &fused_add_rms_norm_splitk_scaled);
  amd.def("rms_norm_fp8(Tensor input, Tensor weight, float epsilon, Tensor q_scale) -> Tensor");
  amd.impl("rms_norm_fp8", torch::kCUDA, &rms_norm_fp8);
  amd.def("fused_add_rms_norm_fp8(Tensor input, Tensor! residual, Tensor weight, float epsilon, Tensor q_scale) -> Tensor");
  amd.impl("fused_add_rms_norm_fp8", torch::kCUDA, &fused_add_rms_norm_fp8);
  amd.def("fused_add_rms_norm_splitk_fp8(Tensor! residual, Tensor partials, Tensor weight, float epsilon, "
          "Tensor? x_scale, Tensor? w_scale, Tensor q_scale) -> Tensor");
  amd.impl("fused_add_rms_norm_splitk_fp8", torch::kCUDA, &fused_add_rms_norm_splitk_fp8);
  amd.def("paged_prefill_workspace_bytes(int num_seqs, int num_tokens, int max_query_len, int num_heads, "
          "int num_kv_heads, int head_size, int max_seq_len) -> int", &paged_prefill_workspace_bytes);
  amd.def("varlen_attention_workspace_bytes(int num_tokens, int num_seqs, int max_seq_len, int num_kv_heads, "
          "int head_size) -> int", &varlen_attention_workspace_bytes);
  amd.def("varlen_attention(Tensor! out, Tensor query, Tensor key, Tensor value, Tensor cu_seqlens, "
          "int max_seq_len, float scale, bool causal, Tensor? alibi_slopes, int sliding_window, "
          "float softcap, Tensor! workspace) -> ()");
  amd.impl("varlen_attention", torch::kCUDA, &varlen_attention);
}


// importable as a Python module (`import light_vllm_amd._C` style), as
// csrc/core/registration.h:18-22 does for the reference's extension
PyMODINIT_FUNC PyInit__C(void) {
  static struct PyModuleDef module = {PyModuleDef_HEAD_INIT, "_C", nullptr, 0, nullptr};
  return PyModule_Create(&module);
}
