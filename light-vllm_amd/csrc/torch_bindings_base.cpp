// torch op registrations of the base library (liblvllm_base.so): what every model of the framework needs -- cache block
// movement, the weight-streaming GEMMs of decode steps, step inputs, the device sampler.  Schemas of the reference's
// operators are its own (csrc/torch_bindings.cpp:18-279); each operator unpacks tensors and forwards to the C-ABI of
// include/lvllm_hip.h on the CURRENT stream of the tensor's device.  Host-only C++ (built with g++).
#include "torch_bindings.h"

namespace {

void swap_blocks(torch::Tensor& src, torch::Tensor& dst, const torch::Tensor& block_mapping) {
  const bool src_dev = src.is_cuda(), dst_dev = dst.is_cuda();
  if (src_dev && dst_dev)
    TORCH_CHECK(src.device().index() == dst.device().index(), "src and dst must be on the same GPU");
  TORCH_CHECK(src_dev || dst_dev, "Invalid device combination");
  TORCH_CHECK(block_mapping.device().is_cpu(), "block_mapping must be on CPU");
  TORCH_CHECK(block_mapping.scalar_type() == at::kLong, "block_mapping must be int64");
  auto bm = block_mapping.contiguous();
  // a block and its padding, if the allocation pads (both sides must pad alike: runs of blocks move as one copy)
  TORCH_CHECK(blocks_are_dense(src) && blocks_are_dense(dst) && src.dim() >= 1 && dst.dim() >= 1 &&
                  src.stride(0) == dst.stride(0) && src.element_size() == dst.element_size(),
              "swap_blocks: src and dst must have dense blocks and the same block stride");
  const int64_t block_bytes = src.element_size() * src.stride(0);
  const torch::Tensor& dev_t = src_dev ? src : dst;
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(dev_t));
  check(lvllm_swap_blocks(src.data_ptr(), dst.data_ptr(), bm.data_ptr<int64_t>(), (int)bm.size(0),
                          block_bytes, src_dev, dst_dev, current_stream(dev_t)));
}

// Device pointer tables for copy_blocks are cached per set of cache tensors, so
// the steady state does no host->device copy and never synchronises (the
// reference re-uploads them on every call, csrc/cache_kernels.cu:128-133).
struct PtrTable {
  std::vector<int64_t> key_ptrs, value_ptrs;
  torch::Tensor dev;  // [2, L] int64 on the cache device
};

void copy_blocks(std::vector<torch::Tensor> const& key_caches,
                 std::vector<torch::Tensor> const& value_caches,
                 const torch::Tensor& block_mapping) {
  const int num_layers = (int)key_caches.size();
  TORCH_CHECK(num_layers == (int)value_caches.size());
  if (num_layers == 0) return;
  const auto dev = key_caches[0].device();
  TORCH_CHECK(dev.is_cuda());
  const int num_pairs = (int)block_mapping.size(0);
  if (num_pairs == 0) return;
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(dev);

  static thread_local PtrTable table;
  std::vector<int64_t> kp(num_layers), vp(num_layers);
  for (int l = 0; l < num_layers; ++l) {
    kp[l] = (int64_t)key_caches[l].data_ptr();
    vp[l] = (int64_t)value_caches[l].data_ptr();
  }
  if (kp != table.key_ptrs || vp != table.value_ptrs || !table.dev.defined() ||
      table.dev.device() != dev) {
    auto host = torch::empty({2, num_layers}, torch::dtype(torch::kInt64));
    for (int l = 0; l < num_layers; ++l) {
      host[0][l] = kp[l];
      host[1][l] = vp[l];
    }
    table.dev = host.to(dev);
    table.key_ptrs = kp;
    table.value_ptrs = vp;
  }
  // the kernel reads block_mapping on the device (csrc/cache_kernels.cu:79-80)
  torch::Tensor bm = block_mapping.to(dev, torch::kInt64, /*non_blocking=*/true).contiguous();
  // (a block and its padding, if the allocation pads: every layer's caches pad alike)
  for (int l = 0; l < num_layers; ++l)
    TORCH_CHECK(blocks_are_dense(key_caches[l]) && blocks_are_dense(value_caches[l]) &&
                    key_caches[l].stride(0) == key_caches[0].stride(0) &&
                    value_caches[l].stride(0) == key_caches[0].stride(0),
                "copy_blocks: dense blocks, one block stride for every cache");
  const int64_t block_bytes = key_caches[0].element_size() * key_caches[0].stride(0);
  const int64_t* base = table.dev.data_ptr<int64_t>();
  check(lvllm_copy_blocks((const void* const*)base, (const void* const*)(base + num_layers),
                          bm.data_ptr<int64_t>(), num_layers, num_pairs, block_bytes,
                          current_stream(key_caches[0])));
}

void reshape_and_cache(torch::Tensor& key, torch::Tensor& value, torch::Tensor& key_cache,
                       torch::Tensor& value_cache, torch::Tensor& slot_mapping,
                       const std::string& kv_cache_dtype, const double k_scale,
                       const double v_scale) {
  LV_CHECK_DEVICE(key);
  TORCH_CHECK(slot_mapping.scalar_type() == at::kLong, "slot_mapping must be int64");
  TORCH_CHECK(blocks_are_dense(key_cache) && blocks_are_dense(value_cache) &&
                  key_cache.stride(0) == value_cache.stride(0),
              "key_cache / value_cache: dense blocks, the same block stride");
  check_cache_dtype(key_cache, key, kv_dtype_code(kv_cache_dtype), "reshape_and_cache");
  check_cache_dtype(value_cache, key, kv_dtype_code(kv_cache_dtype), "reshape_and_cache");
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(key));
  check(lvllm_reshape_and_cache_strided(key.data_ptr(), value.data_ptr(), key_cache.data_ptr(),
                                        value_cache.data_ptr(), slot_mapping.data_ptr<int64_t>(),
                                        (int)key.size(0), (int)key.size(1), (int)key.size(2),
                                        (int)key_cache.size(3), (int)key_cache.size(4), key.stride(0),
                                        value.stride(0), dtype_code(key, "reshape_and_cache"),
                                        kv_dtype_code(kv_cache_dtype), (float)k_scale, (float)v_scale,
                                        cache_extent_bytes(key_cache, value_cache), key_cache.stride(0),
                                        current_stream(key)));
}

void reshape_and_cache_flash(torch::Tensor& key, torch::Tensor& value, torch::Tensor& key_cache,
                             torch::Tensor& value_cache, torch::Tensor& slot_mapping,
                             const std::string& kv_cache_dtype, const double k_scale,
                             const double v_scale) {
  LV_CHECK_DEVICE(key);
  TORCH_CHECK(slot_mapping.scalar_type() == at::kLong, "slot_mapping must be int64");
  TORCH_CHECK(key_cache.stride(0) == value_cache.stride(0));
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(key));
  check(lvllm_reshape_and_cache_flash(
      key.data_ptr(), value.data_ptr(), key_cache.data_ptr(), value_cache.data_ptr(),
      slot_mapping.data_ptr<int64_t>(), (int)key.size(0), (int)key.size(1), (int)key.size(2),
      (int)key_cache.size(1), key_cache.stride(0), key.stride(0), value.stride(0),
      dtype_code(key, "reshape_and_cache_flash"), kv_dtype_code(kv_cache_dtype), (float)k_scale,
      (float)v_scale, current_stream(key)));
}

// Extension ops (not in the reference): F.linear for decode batches through the
// weight-streaming kernel.  `packed_shape` = [N, K] when `w` is in lvllm_pack_weight order.
torch::Tensor skinny_linear_impl(const torch::Tensor& x, const torch::Tensor& w,
                                 const std::optional<torch::Tensor>& bias, bool packed, int64_t N,
                                 int64_t K) {
  const int64_t M = x.size(0);
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(x));
  auto y = torch::empty({M, N}, x.options());
  const int64_t ws_bytes = lvllm_skinny_gemm_workspace_bytes((int)M, (int)N, (int)K);
  torch::Tensor ws;
  if (ws_bytes > 0) ws = torch::empty({ws_bytes / 4}, x.options().dtype(torch::kFloat));
  const int rc = lvllm_skinny_gemm(y.data_ptr(), x.data_ptr(), w.data_ptr(), bias ? bias->data_ptr() : nullptr,
                                   (int)M, (int)N, (int)K, x.stride(0), dtype_code(x, "skinny_linear"),
                                   packed ? 1 : 0, ws_bytes > 0 ? ws.data_ptr() : nullptr, ws_bytes,
                                   current_stream(x));
  if (rc == 3) return torch::Tensor();  // outside the envelope
  check(rc);
  return y;
}

bool skinny_ok(const torch::Tensor& x, const torch::Tensor& w, const std::optional<torch::Tensor>& bias) {
  return x.is_cuda() && x.dim() == 2 && (x.scalar_type() == at::kBFloat16 || x.scalar_type() == at::kHalf) &&
         w.scalar_type() == x.scalar_type() && w.is_contiguous() && x.stride(1) == 1 && x.size(0) <= 64 &&
         x.size(0) > 0 && (!bias || bias->is_contiguous());
}

torch::Tensor skinny_linear(const torch::Tensor& x, const torch::Tensor& w,
                            const std::optional<torch::Tensor>& bias) {
  TORCH_CHECK(x.dim() == 2 && w.dim() == 2 && x.size(1) == w.size(1), "skinny_linear: x [M,K], w [N,K]");
  if (skinny_ok(x, w, bias)) {
    auto y = skinny_linear_impl(x, w, bias, false, w.size(0), w.size(1));
    if (y.defined()) return y;
  }
  return at::linear(x, w, bias);
}

torch::Tensor skinny_linear_packed(const torch::Tensor& x, const torch::Tensor& w_packed,
                                   const std::optional<torch::Tensor>& bias, int64_t N, int64_t K) {
  TORCH_CHECK(x.dim() == 2 && x.size(1) == K && w_packed.numel() == N * K, "skinny_linear_packed: bad shapes");
  TORCH_CHECK(skinny_ok(x, w_packed, bias), "skinny_linear_packed: M <= 64 rows of bf16/f16 on the GPU only");
  auto y = skinny_linear_impl(x, w_packed, bias, true, N, K);
  TORCH_CHECK(y.defined(), lvllm_last_error());
  return y;
}

// lm_head + greedy sampling: int64 [M] = argmax(x . w^T) over the rounded values, no logits tensor (in the
// projection's epilogue, or inside its split-K reduce pass when K is split over workgroups at this M).
torch::Tensor skinny_linear_packed_argmax(const torch::Tensor& x, const torch::Tensor& w_packed, int64_t N, int64_t K) {
  TORCH_CHECK(x.dim() == 2 && x.size(1) == K && w_packed.numel() == N * K, "skinny_linear_packed_argmax: bad shapes");
  TORCH_CHECK(skinny_ok(x, w_packed, std::nullopt), "skinny_linear_packed_argmax: M <= 64 rows of bf16/f16 on the GPU only");
  const int64_t M = x.size(0);
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(x));
  auto tokens = torch::empty({M}, x.options().dtype(torch::kLong));
  const int64_t ws_bytes = lvllm_skinny_gemm_argmax_workspace_bytes_ex((int)M, (int)N, (int)K);
  auto ws = torch::empty({ws_bytes / 4}, x.options().dtype(torch::kFloat));
  check(lvllm_skinny_gemm_argmax(tokens.data_ptr<int64_t>(), x.data_ptr(), w_packed.data_ptr(), (int)M, (int)N, (int)K,
                                 x.stride(0), dtype_code(x, "skinny_linear_packed_argmax"), ws.data_ptr(), ws_bytes,
                                 current_stream(x)));
  return tokens;
}

// 65..256 rows (large decode batches, prefill chunks): X through LDS, see lvllm_stream_gemm
torch::Tensor stream_linear_packed(const torch::Tensor& x, const torch::Tensor& w_packed,
                                   const std::optional<torch::Tensor>& bias, int64_t N, int64_t K) {
  TORCH_CHECK(x.dim() == 2 && x.size(1) == K && w_packed.numel() == N * K && x.stride(1) == 1,
              "stream_linear_packed: bad shapes");
  TORCH_CHECK(x.is_cuda() && w_packed.is_cuda() && w_packed.is_contiguous() && x.size(0) >= 1 && x.size(0) <= 256 &&
                  (x.scalar_type() == at::kBFloat16 || x.scalar_type() == at::kHalf) &&
                  w_packed.scalar_type() == x.scalar_type() && (!bias || bias->is_contiguous()),
              "stream_linear_packed: 1..256 rows of bf16/f16 on the GPU");
  const int64_t M = x.size(0);
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(x));
  auto y = torch::empty({M, N}, x.options());
  const int64_t ws_bytes = lvllm_stream_gemm_workspace_bytes((int)M, (int)N, (int)K);
  torch::Tensor ws;
  if (ws_bytes > 0) ws = torch::empty({ws_bytes / 4}, x.options().dtype(torch::kFloat));
  check(lvllm_stream_gemm(y.data_ptr(), x.data_ptr(), w_packed.data_ptr(), bias ? bias->data_ptr() : nullptr, (int)M,
                          (int)N, (int)K, x.stride(0), dtype_code(x, "stream_linear_packed"),
                          ws_bytes > 0 ? ws.data_ptr() : nullptr, ws_bytes, current_stream(x)));
  return y;
}

// gate_up projection + silu_and_mul in one launch: w_packed holds [gate rows | up rows] ([N, K]
// packed), the result is [M, N / 2].  Bit-identical to skinny_linear_packed followed by silu_and_mul.
torch::Tensor skinny_linear_packed_swiglu(const torch::Tensor& x, const torch::Tensor& w_packed,
                                          const std::optional<torch::Tensor>& bias, int64_t N, int64_t K) {
  TORCH_CHECK(x.dim() == 2 && x.size(1) == K && w_packed.numel() == N * K && N % 32 == 0,
              "skinny_linear_packed_swiglu: bad shapes");
  TORCH_CHECK(skinny_ok(x, w_packed, bias), "skinny_linear_packed_swiglu: M <= 64 rows of bf16/f16 on the GPU only");
  const int64_t M = x.size(0);
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(x));
  auto y = torch::empty({M, N / 2}, x.options());
  // K split over workgroups at this M: the fp32 partials are summed and activated by one reduce launch
  const int64_t ws_bytes = lvllm_skinny_gemm_workspace_bytes((int)M, (int)N, (int)K);
  torch::Tensor ws;
  if (ws_bytes > 0) ws = torch::empty({ws_bytes / 4}, x.options().dtype(torch::kFloat));
  check(lvllm_skinny_gemm_ex(y.data_ptr(), x.data_ptr(), w_packed.data_ptr(), bias ? bias->data_ptr() : nullptr,
                             (int)M, (int)N, (int)K, x.stride(0), dtype_code(x, "skinny_linear_packed_swiglu"), 1, 2,
                             0, nullptr, ws_bytes > 0 ? ws.data_ptr() : nullptr, ws_bytes, current_stream(x)));
  return y;
}

// y = max(x . w^T, 0)^2: the squared-ReLU feed-forward's up projection in one launch, bit-identical to the two
torch::Tensor skinny_linear_packed_relu_squared(const torch::Tensor& x, const torch::Tensor& w_packed, int64_t N, int64_t K) {
  TORCH_CHECK(x.dim() == 2 && x.size(1) == K && w_packed.numel() == N * K, "skinny_linear_packed_relu_squared: bad shapes");
  TORCH_CHECK(skinny_ok(x, w_packed, std::nullopt),
              "skinny_linear_packed_relu_squared: M <= 64 rows of bf16/f16 on the GPU only");
  const int64_t M = x.size(0);
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(x));
  auto y = torch::empty({M, N}, x.options());
  const int64_t ws_bytes = lvllm_skinny_gemm_workspace_bytes((int)M, (int)N, (int)K);
  torch::Tensor ws;
  if (ws_bytes > 0) ws = torch::empty({ws_bytes / 4}, x.options().dtype(torch::kFloat));
  check(lvllm_skinny_gemm_ex(y.data_ptr(), x.data_ptr(), w_packed.data_ptr(), nullptr, (int)M, (int)N, (int)K, x.stride(0),
                             dtype_code(x, "skinny_linear_packed_relu_squared"), 1, 5, 0, nullptr,
                             ws_bytes > 0 ? ws.data_ptr() : nullptr, ws_bytes, current_stream(x)));
  return y;
}

// The clamped unit of a feed-forward's gate and up projection, [gate rows | up rows], in one launch: clamped_unit of the plain
// projection
torch::Tensor skinny_linear_packed_clamped_unit(const torch::Tensor& x, const torch::Tensor& w_packed, int64_t N, int64_t K,
                                                double limit) {
  const char* op = "skinny_linear_packed_clamped_unit";
  TORCH_CHECK(x.dim() == 2 && x.size(1) == K && w_packed.numel() == N * K && N % 32 == 0, op, ": bad shapes");
  TORCH_CHECK(skinny_ok(x, w_packed, std::nullopt), op, ": M <= 64 rows of bf16/f16 on the GPU only");
  const int64_t M = x.size(0);
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(x));
  auto y = torch::empty({M, N / 2}, x.options());
  const int64_t ws_bytes = lvllm_skinny_gemm_workspace_bytes((int)M, (int)N, (int)K);
  torch::Tensor ws;
  if (ws_bytes > 0) ws = torch::empty({ws_bytes / 4}, x.options().dtype(torch::kFloat));
  check(lvllm_skinny_gemm_clamped_unit(y.data_ptr(), x.data_ptr(), w_packed.data_ptr(), (int)M, (int)N, (int)K, x.stride(0),
                                       dtype_code(x, op), 1, (float)limit, ws_bytes > 0 ? ws.data_ptr() : nullptr, ws_bytes,
                                       current_stream(x)));
  return y;
}

// silu(gate) * up of [rows, gate | up]
torch::Tensor silu_unit(const torch::Tensor& x) {
  const char* op = "silu_unit";
  LV_CHECK_DEVICE(x);
  TORCH_CHECK(x.dim() == 2 && x.is_contiguous() && x.size(1) % 2 == 0, op, ": contiguous [rows, gate | up]");
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(x));
  auto y = torch::empty({x.size(0), x.size(1) / 2}, x.options());
  check(lvllm_silu_and_mul(y.data_ptr(), x.data_ptr(), x.size(0), (int)y.size(1), dtype_code(x, op), current_stream(x)));
  return y;
}

torch::Tensor clamped_unit(const torch::Tensor& x, double limit) {
  const char* op = "clamped_unit";
  LV_CHECK_DEVICE(x);
  TORCH_CHECK(x.dim() == 2 && x.is_contiguous() && x.size(1) % 2 == 0, op, ": contiguous [rows, gate | up]");
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(x));
  auto y = torch::empty({x.size(0), x.size(1) / 2}, x.options());
  check(lvllm_clamped_unit(y.data_ptr(), x.data_ptr(), x.size(0), (int)y.size(1), (float)limit, dtype_code(x, op),
                           current_stream(x)));
  return y;
}

// A projection that leaves its fp32 split-K partials [S, M, N] for fused_add_rms_norm_splitk
// instead of reducing them itself.  swiglu: x = [gate | up] ([M, 2K]) and the activation is applied
// while loading x (bit-identical to silu_and_mul, but every workgroup redoes it for its K slice:
// measured 2x slower than the separate activation kernel at inter=14336 -- kept for small shapes).
torch::Tensor skinny_linear_packed_partials(const torch::Tensor& gate_up, const torch::Tensor& w_packed, int64_t N,
                                            int64_t K, bool swiglu) {
  TORCH_CHECK(gate_up.dim() == 2 && gate_up.size(1) == (swiglu ? 2 * K : K) && w_packed.numel() == N * K,
              "bad shapes");
  TORCH_CHECK(skinny_ok(gate_up, w_packed, std::nullopt), "M <= 64 rows of bf16/f16 on the GPU only");
  const int64_t M = gate_up.size(0);
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(gate_up));
  int64_t ws_bytes = lvllm_skinny_gemm_workspace_bytes((int)M, (int)N, (int)K);
  if (ws_bytes == 0) ws_bytes = M * N * 4;
  int64_t S = ws_bytes / (M * N * 4);
  if (S < 16) S = 16;  // room for a forced finer split (tuning "gemm_partials_ksplit"); the slabs used are returned
  ws_bytes = S * M * N * 4;
  auto partials = torch::empty({S, M, N}, gate_up.options().dtype(torch::kFloat));
  int ksplit = 0;
  check(lvllm_skinny_gemm_ex(nullptr, gate_up.data_ptr(), w_packed.data_ptr(), nullptr, (int)M, (int)N, (int)K,
                             gate_up.stride(0), dtype_code(gate_up, "skinny_linear_packed_partials"), 1,
                             swiglu ? 1 : 0, 1, &ksplit,
                             partials.data_ptr(), ws_bytes, current_stream(gate_up)));
  TORCH_CHECK(ksplit >= 1 && ksplit <= S, "split count mismatch");
  return ksplit == S ? partials : partials.narrow(0, 0, ksplit);
}

// A W8A8 projection whose K is split over workgroups, leaving the raw fp32 partials [S, M, N] for
// fused_add_rms_norm_splitk_scaled.  Returns an EMPTY tensor when K is not split at this shape (nothing was done).
torch::Tensor skinny_linear_w8a8_partials(const torch::Tensor& x, const torch::Tensor& w_packed,
                                          const torch::Tensor& w_scale, const torch::Tensor& x_scale, int64_t N,
                                          int64_t K) {
  TORCH_CHECK(x.dim() == 2 && x.size(1) == K && x.is_cuda() && x.stride(1) == 1, "bad x");
  const int64_t M = x.size(0);
  const int64_t ws_bytes = lvllm_skinny_gemm_w8a8_workspace_bytes((int)M, (int)N, (int)K);
  if (ws_bytes == 0 || M == 0) return torch::empty({0}, x.options().dtype(torch::kFloat));
  const int64_t S = ws_bytes / (M * N * 4);
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(x));
  auto partials = torch::empty({S, M, N}, x.options().dtype(torch::kFloat));
  const int rc = lvllm_skinny_gemm_w8a8_ex(nullptr, x.data_ptr(), w_packed.data_ptr(), nullptr,
                                           x_scale.data_ptr<float>(), w_scale.data_ptr<float>(), (int)M, (int)N,
                                           (int)K, x.stride(0), dtype_code(x, "skinny_linear_w8a8_partials"), 4,
                                           partials.data_ptr(), ws_bytes, current_stream(x));
  if (rc == 3) return torch::empty({0}, x.options().dtype(torch::kFloat));
  check(rc);
  return partials;
}

// csrc/prepare_inputs/advance_step.cu:59-125: same argument checks (verify_tensor)
void advance_step(int64_t num_seqs, int64_t num_queries, int64_t block_size, torch::Tensor& input_tokens,
                  torch::Tensor& sampled_token_ids, torch::Tensor& input_positions, torch::Tensor& seq_lens,
                  torch::Tensor& slot_mapping, torch::Tensor& block_tables) {
  auto verify = [](const char* name, const torch::Tensor& t, int64_t size_0, int64_t size_1, c10::ScalarType type) {
    const bool ok = (size_0 == -1 || t.size(0) == size_0) && (size_1 == -1 || (t.dim() > 1 && t.size(1) == size_1)) &&
                    t.is_contiguous() && t.scalar_type() == type && t.is_cuda();
    TORCH_CHECK(ok, "tensor: name = ", name, ", shape = ", t.sizes(), " is_cont = ", t.is_contiguous(),
                ", type = ", t.dtype(), " is not as expected: shape = [", size_0, ", ", size_1, "], type = ", type);
  };
  verify("input_tokens", input_tokens, num_seqs, -1, at::kLong);
  verify("sampled_token_ids", sampled_token_ids, num_queries, 1, at::kLong);
  verify("input_positions", input_positions, num_seqs, -1, at::kLong);
  verify("seq_lens", seq_lens, num_seqs, -1, at::kInt);
  verify("slot_mapping", slot_mapping, num_seqs, -1, at::kLong);
  verify("block_tables", block_tables, num_seqs, -1, at::kInt);
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(sampled_token_ids));
  check(lvllm_advance_step((int)num_seqs, (int)num_queries, (int)block_size, input_tokens.data_ptr<int64_t>(),
                           sampled_token_ids.data_ptr<int64_t>(), input_positions.data_ptr<int64_t>(),
                           seq_lens.data_ptr<int32_t>(), slot_mapping.data_ptr<int64_t>(),
                           block_tables.data_ptr<int32_t>(), block_tables.stride(0),
                           current_stream(sampled_token_ids)));
}

// Extension: advance_step between the model steps of a multi-step decode.  Same arithmetic; the sampled
// ids are also logged into `token_log` and rows of the padded batch without a sequence are skipped.
void advance_step_logged(int64_t block_size, torch::Tensor& input_tokens, const torch::Tensor& sampled_token_ids,
                         torch::Tensor& input_positions, torch::Tensor& seq_lens, torch::Tensor& slot_mapping,
                         const torch::Tensor& block_tables, torch::Tensor& token_log) {
  const int64_t n = input_tokens.size(0);
  TORCH_CHECK(input_tokens.is_cuda() && input_tokens.scalar_type() == at::kLong && input_tokens.is_contiguous());
  TORCH_CHECK(sampled_token_ids.scalar_type() == at::kLong && sampled_token_ids.is_contiguous() &&
              sampled_token_ids.numel() >= n);
  TORCH_CHECK(input_positions.scalar_type() == at::kLong && input_positions.is_contiguous() && input_positions.size(0) == n);
  TORCH_CHECK(seq_lens.scalar_type() == at::kInt && seq_lens.is_contiguous() && seq_lens.size(0) == n);
  TORCH_CHECK(slot_mapping.scalar_type() == at::kLong && slot_mapping.is_contiguous() && slot_mapping.size(0) == n);
  TORCH_CHECK(block_tables.scalar_type() == at::kInt && block_tables.dim() == 2 && block_tables.size(0) == n &&
              block_tables.stride(1) == 1);
  TORCH_CHECK(token_log.scalar_type() == at::kLong && token_log.is_contiguous() && token_log.numel() >= n);
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(input_tokens));
  check(lvllm_advance_step_ex((int)n, (int)n, (int)block_size, input_tokens.data_ptr<int64_t>(),
                              sampled_token_ids.data_ptr<int64_t>(), input_positions.data_ptr<int64_t>(),
                              seq_lens.data_ptr<int32_t>(), slot_mapping.data_ptr<int64_t>(),
                              block_tables.data_ptr<int32_t>(), block_tables.stride(0),
                              token_log.data_ptr<int64_t>(), 1, current_stream(input_tokens)));
}

// Device-side sampler (include/lvllm_hip.h: lvllm_sample_rows).  `params` uint8 [num_slots, 128], `counts` int32
// [num_slots, vocab], `scratch` float [rows, >= vocab]; all three absent = every row plain greedy.
void sample_rows(torch::Tensor& tokens_out, const torch::Tensor& logits, const std::optional<torch::Tensor>& state_slot,
                 const std::optional<torch::Tensor>& params, const std::optional<torch::Tensor>& counts,
                 const std::optional<torch::Tensor>& scratch, const std::optional<torch::Tensor>& processed_out,
                 bool update_state) {
  LV_CHECK_DEVICE(logits);
  TORCH_CHECK(logits.dim() == 2 && logits.stride(1) == 1, "sample_rows: logits [rows, vocab], unit inner stride");
  const int64_t rows = logits.size(0), vocab = logits.size(1);
  TORCH_CHECK(tokens_out.is_cuda() && tokens_out.scalar_type() == at::kLong && tokens_out.is_contiguous() &&
              tokens_out.numel() >= rows, "sample_rows: tokens_out int64 [rows]");
  const int32_t* slot = nullptr;
  void* pp = nullptr;
  int32_t* cc = nullptr;
  float* sc = nullptr;
  float* po = nullptr;
  int64_t cstride = 0, sstride = 0, pstride = 0, nslots = 0;
  if (state_slot.has_value()) {
    TORCH_CHECK(params.has_value() && counts.has_value() && scratch.has_value(),
                "sample_rows: state_slot needs params, counts and scratch");
    TORCH_CHECK(state_slot->is_cuda() && state_slot->scalar_type() == at::kInt && state_slot->is_contiguous() &&
                state_slot->numel() >= rows, "sample_rows: state_slot int32 [rows]");
    TORCH_CHECK(params->is_cuda() && params->scalar_type() == at::kByte && params->is_contiguous() && params->dim() == 2 &&
                params->size(1) == LVLLM_SAMPLER_PARAMS_BYTES, "sample_rows: params uint8 [slots, 128]");
    TORCH_CHECK(counts->is_cuda() && counts->scalar_type() == at::kInt && counts->dim() == 2 && counts->stride(1) == 1 &&
                counts->size(0) == params->size(0) && counts->size(1) >= vocab, "sample_rows: counts int32 [slots, vocab]");
    TORCH_CHECK(scratch->is_cuda() && scratch->scalar_type() == at::kFloat && scratch->dim() == 2 &&
                scratch->stride(1) == 1 && scratch->size(0) >= rows && scratch->size(1) >= vocab,
                "sample_rows: scratch float [rows, >= vocab]");
    slot = state_slot->data_ptr<int32_t>();
    pp = params->data_ptr();
    cc = counts->data_ptr<int32_t>();
    sc = scratch->data_ptr<float>();
    cstride = counts->stride(0);
    sstride = scratch->stride(0);
    nslots = params->size(0);
  }
  if (processed_out.has_value()) {
    TORCH_CHECK(processed_out->is_cuda() && processed_out->scalar_type() == at::kFloat && processed_out->dim() == 2 &&
                processed_out->stride(1) == 1 && processed_out->size(0) >= rows && processed_out->size(1) >= vocab,
                "sample_rows: processed_out float [rows, >= vocab]");
    po = processed_out->data_ptr<float>();
    pstride = processed_out->stride(0);
  }
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(logits));
  check(lvllm_sample_rows(tokens_out.data_ptr<int64_t>(), logits.data_ptr(), logits.stride(0),
                          dtype_code(logits, "sample_rows"), (int)rows, (int)vocab, slot, pp, cc, cstride, (int)nslots, sc,
                          sstride, po, pstride, update_state ? 1 : 0, current_stream(logits)));
}

void sampler_init_row(torch::Tensor& counts_row, const torch::Tensor& prompt_tokens, const torch::Tensor& output_tokens) {
  LV_CHECK_DEVICE(counts_row);
  TORCH_CHECK(counts_row.scalar_type() == at::kInt && counts_row.dim() == 1 && counts_row.stride(0) == 1);
  TORCH_CHECK(prompt_tokens.is_cuda() && prompt_tokens.scalar_type() == at::kLong && prompt_tokens.is_contiguous());
  TORCH_CHECK(output_tokens.is_cuda() && output_tokens.scalar_type() == at::kLong && output_tokens.is_contiguous());
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(counts_row));
  check(lvllm_sampler_init_row(counts_row.data_ptr<int32_t>(), (int)counts_row.size(0), prompt_tokens.data_ptr<int64_t>(),
                               (int)prompt_tokens.numel(), output_tokens.data_ptr<int64_t>(), (int)output_tokens.numel(),
                               current_stream(counts_row)));
}

// csrc/cache_kernels.cu:352-410
void convert_fp8(torch::Tensor& dst_cache, torch::Tensor& src_cache, const double scale,
                 const std::string& kv_cache_dtype) {
  TORCH_CHECK(src_cache.is_cuda(), "src must be on a GPU");
  TORCH_CHECK(dst_cache.is_cuda(), "dst must be on a GPU");
  TORCH_CHECK(src_cache.device().index() == dst_cache.device().index(), "src and dst must be on the same GPU");
  TORCH_CHECK(src_cache.is_contiguous() && dst_cache.is_contiguous() && src_cache.numel() == dst_cache.numel(),
              "convert_fp8: contiguous tensors of equal size");
  TORCH_CHECK(kv_cache_dtype == "fp8" || kv_cache_dtype == "fp8_e4m3", "Unsupported data type: ", kv_cache_dtype);
  const bool to_fp8 = dst_cache.element_size() == 1;
  TORCH_CHECK(to_fp8 != (src_cache.element_size() == 1), "convert_fp8: exactly one side must be a one-byte tensor");
  const torch::Tensor& wide = to_fp8 ? src_cache : dst_cache;
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(src_cache));
  check(lvllm_convert_fp8(dst_cache.data_ptr(), src_cache.data_ptr(), (float)scale, src_cache.numel(),
                          dtype_code(wide, "convert_fp8"), to_fp8 ? 1 : 0, LVLLM_KV_FP8_E4M3,
                          current_stream(src_cache)));
}

torch::Tensor skinny_linear_w8a8(const torch::Tensor& x, const torch::Tensor& w_packed, const torch::Tensor& w_scale,
                                 const torch::Tensor& x_scale, int64_t N, int64_t K,
                                 const std::optional<torch::Tensor>& bias) {
  LV_CHECK_DEVICE(x);
  LV_CHECK_DEVICE(w_packed);
  TORCH_CHECK(x.dim() == 2 && x.size(1) == K && x.stride(1) == 1, "skinny_linear_w8a8: x must be [M, K]");
  TORCH_CHECK(w_packed.is_contiguous() && w_packed.numel() * w_packed.element_size() == N * K,
              "skinny_linear_w8a8: w_packed must hold N*K fp8 bytes");
  TORCH_CHECK(w_scale.scalar_type() == at::kFloat && x_scale.scalar_type() == at::kFloat && w_scale.is_cuda() &&
                  x_scale.is_cuda() && w_scale.numel() == 1 && x_scale.numel() == 1,
              "skinny_linear_w8a8: per-tensor float32 scales on the device");
  const int64_t M = x.size(0);
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(x));
  auto y = torch::empty({M, N}, x.options());
  const int64_t ws_bytes = lvllm_skinny_gemm_w8a8_workspace_bytes((int)M, (int)N, (int)K);
  torch::Tensor ws;
  if (ws_bytes > 0) ws = torch::empty({ws_bytes / 4}, x.options().dtype(torch::kFloat));
  check(lvllm_skinny_gemm_w8a8(y.data_ptr(), x.data_ptr(), w_packed.data_ptr(), bias ? bias->data_ptr() : nullptr,
                               x_scale.data_ptr<float>(), w_scale.data_ptr<float>(), (int)M, (int)N, (int)K,
                               x.stride(0), dtype_code(x, "skinny_linear_w8a8"),
                               ws_bytes > 0 ? ws.data_ptr() : nullptr, ws_bytes, current_stream(x)));
  return y;
}

// W8A8 gate_up projection + silu_and_mul in one launch ([M, N / 2]); falls back to the two launches
// when K is split over workgroups at this M.  Bit-identical to skinny_linear_w8a8 + silu_and_mul.
torch::Tensor skinny_linear_w8a8_swiglu(const torch::Tensor& x, const torch::Tensor& w_packed,
                                        const torch::Tensor& w_scale, const torch::Tensor& x_scale, int64_t N,
                                        int64_t K, const std::optional<torch::Tensor>& bias) {
  TORCH_CHECK(N % 32 == 0, "skinny_linear_w8a8_swiglu: N must be a multiple of 32");
  const int64_t M = x.size(0);
  auto y = torch::empty({M, N / 2}, x.options());
  if (lvllm_skinny_gemm_w8a8_workspace_bytes((int)M, (int)N, (int)K) > 0) {
    auto gate_up = skinny_linear_w8a8(x, w_packed, w_scale, x_scale, N, K, bias);
    const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(x));
    check(lvllm_silu_and_mul(y.data_ptr(), gate_up.data_ptr(), M, (int)(N / 2), dtype_code(x, "silu_and_mul"),
                             current_stream(x)));
    return y;
  }
  LV_CHECK_DEVICE(x);
  LV_CHECK_DEVICE(w_packed);
  TORCH_CHECK(x.dim() == 2 && x.size(1) == K && x.stride(1) == 1, "skinny_linear_w8a8_swiglu: x must be [M, K]");
  TORCH_CHECK(w_packed.is_contiguous() && w_packed.numel() * w_packed.element_size() == N * K,
              "skinny_linear_w8a8_swiglu: w_packed must hold N*K fp8 bytes");
  TORCH_CHECK(w_scale.scalar_type() == at::kFloat && x_scale.scalar_type() == at::kFloat && w_scale.is_cuda() &&
                  x_scale.is_cuda() && w_scale.numel() == 1 && x_scale.numel() == 1,
              "skinny_linear_w8a8_swiglu: per-tensor float32 scales on the device");
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(x));
  check(lvllm_skinny_gemm_w8a8_ex(y.data_ptr(), x.data_ptr(), w_packed.data_ptr(), bias ? bias->data_ptr() : nullptr,
                                  x_scale.data_ptr<float>(), w_scale.data_ptr<float>(), (int)M, (int)N, (int)K,
                                  x.stride(0), dtype_code(x, "skinny_linear_w8a8_swiglu"), 2, nullptr, 0,
                                  current_stream(x)));
  return y;
}

static void check_w8a8_q(const torch::Tensor& x8, const torch::Tensor& w_packed, const torch::Tensor& w_scale,
                         const torch::Tensor& x_scale, int64_t N, int64_t K, const char* op) {
  LV_CHECK_DEVICE(x8);
  LV_CHECK_DEVICE(w_packed);
  TORCH_CHECK(x8.dim() == 2 && x8.size(1) == K && x8.stride(1) == 1 && x8.element_size() == 1 && x8.size(0) <= 32, op,
              ": x_fp8 must be [M <= 32, K] bytes");
  TORCH_CHECK(w_packed.is_contiguous() && w_packed.numel() * w_packed.element_size() == N * K, op,
              ": w_packed must hold N*K fp8 bytes");
  check_q_scale(w_scale, op);
  check_q_scale(x_scale, op);
}

// y [M, N] in `out_dtype` = the projection of pre-quantised activations (skinny_linear_w8a8 on the unquantised x)
torch::Tensor skinny_linear_w8a8_q(const torch::Tensor& x8, const torch::Tensor& w_packed, const torch::Tensor& w_scale,
                                   const torch::Tensor& x_scale, int64_t N, int64_t K,
                                   const std::optional<torch::Tensor>& bias, at::ScalarType out_dtype) {
  check_w8a8_q(x8, w_packed, w_scale, x_scale, N, K, "skinny_linear_w8a8_q");
  const int64_t M = x8.size(0);
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(x8));
  auto y = torch::empty({M, N}, x8.options().dtype(out_dtype));
  const int64_t ws_bytes = lvllm_skinny_gemm_w8a8_workspace_bytes((int)M, (int)N, (int)K);
  torch::Tensor ws;
  if (ws_bytes > 0) ws = torch::empty({ws_bytes / 4}, x8.options().dtype(torch::kFloat));
  check(lvllm_skinny_gemm_w8a8_q(y.data_ptr(), nullptr, nullptr, x8.data_ptr(), w_packed.data_ptr(),
                                 bias ? bias->data_ptr() : nullptr, x_scale.data_ptr<float>(), w_scale.data_ptr<float>(),
                                 (int)M, (int)N, (int)K, x8.stride(0), dtype_code(y, "skinny_linear_w8a8_q"), 0,
                                 ws_bytes > 0 ? ws.data_ptr() : nullptr, ws_bytes, current_stream(x8)));
  return y;
}

// the gate_up projection + silu_and_mul + static_scaled_fp8_quant(act, q_scale) in one launch: fp8 [M, N / 2]
torch::Tensor skinny_linear_w8a8_q_swiglu_fp8(const torch::Tensor& x8, const torch::Tensor& w_packed,
                                              const torch::Tensor& w_scale, const torch::Tensor& x_scale, int64_t N,
                                              int64_t K, const torch::Tensor& q_scale, at::ScalarType compute_dtype) {
  check_w8a8_q(x8, w_packed, w_scale, x_scale, N, K, "skinny_linear_w8a8_q_swiglu_fp8");
  check_q_scale(q_scale, "skinny_linear_w8a8_q_swiglu_fp8");
  TORCH_CHECK(N % 32 == 0 && lvllm_skinny_gemm_w8a8_workspace_bytes((int)x8.size(0), (int)N, (int)K) == 0,
              "skinny_linear_w8a8_q_swiglu_fp8: N % 32 == 0 and K within one workgroup");
  const int64_t M = x8.size(0);
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(x8));
  auto y8 = torch::empty({M, N / 2}, x8.options().dtype(torch::kUInt8));
  const int dt = compute_dtype == at::kBFloat16 ? LVLLM_BF16 : LVLLM_F16;
  TORCH_CHECK(compute_dtype == at::kBFloat16 || compute_dtype == at::kHalf, "compute_dtype: bfloat16 or float16");
  check(lvllm_skinny_gemm_w8a8_q(nullptr, y8.data_ptr(), q_scale.data_ptr<float>(), x8.data_ptr(), w_packed.data_ptr(),
                                 nullptr, x_scale.data_ptr<float>(), w_scale.data_ptr<float>(), (int)M, (int)N, (int)K,
                                 x8.stride(0), dt, 2, nullptr, 0, current_stream(x8)));
  return y8;
}

// raw fp32 split-K partials [S, M, N] of a projection of pre-quantised activations (empty: K is not split here)
torch::Tensor skinny_linear_w8a8_q_partials(const torch::Tensor& x8, const torch::Tensor& w_packed,
                                            const torch::Tensor& w_scale, const torch::Tensor& x_scale, int64_t N,
                                            int64_t K) {
  check_w8a8_q(x8, w_packed, w_scale, x_scale, N, K, "skinny_linear_w8a8_q_partials");
  const int64_t M = x8.size(0);
  const int64_t ws_bytes = lvllm_skinny_gemm_w8a8_workspace_bytes((int)M, (int)N, (int)K);
  if (ws_bytes == 0 || M == 0) return torch::empty({0}, x8.options().dtype(torch::kFloat));
  const int64_t S = ws_bytes / (M * N * 4);
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(x8));
  auto partials = torch::empty({S, M, N}, x8.options().dtype(torch::kFloat));
  check(lvllm_skinny_gemm_w8a8_q(nullptr, nullptr, nullptr, x8.data_ptr(), w_packed.data_ptr(), nullptr,
                                 x_scale.data_ptr<float>(), w_scale.data_ptr<float>(), (int)M, (int)N, (int)K,
                                 x8.stride(0), LVLLM_BF16, 4, partials.data_ptr(), ws_bytes, current_stream(x8)));
  return partials;
}

// W8A8 lm_head + greedy sampling in one launch (see skinny_linear_packed_argmax)
torch::Tensor skinny_linear_w8a8_argmax(const torch::Tensor& x, const torch::Tensor& w_packed, const torch::Tensor& w_scale,
                                        const torch::Tensor& x_scale, int64_t N, int64_t K) {
  const int64_t M = x.size(0);
  if (M > 32 || lvllm_skinny_gemm_w8a8_workspace_bytes((int)M, (int)N, (int)K) > 0)  // outside the epilogue's envelope
    return at::argmax(skinny_linear_w8a8(x, w_packed, w_scale, x_scale, N, K, std::nullopt), -1);
  LV_CHECK_DEVICE(x);
  LV_CHECK_DEVICE(w_packed);
  TORCH_CHECK(x.dim() == 2 && x.size(1) == K && x.stride(1) == 1 && M >= 1 && M <= 64,
              "skinny_linear_w8a8_argmax: x must be [M <= 64, K]");
  TORCH_CHECK(w_packed.is_contiguous() && w_packed.numel() * w_packed.element_size() == N * K,
              "skinny_linear_w8a8_argmax: w_packed must hold N*K fp8 bytes");
  TORCH_CHECK(w_scale.scalar_type() == at::kFloat && x_scale.scalar_type() == at::kFloat && w_scale.is_cuda() &&
                  x_scale.is_cuda() && w_scale.numel() == 1 && x_scale.numel() == 1,
              "skinny_linear_w8a8_argmax: per-tensor float32 scales on the device");
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(x));
  auto tokens = torch::empty({M}, x.options().dtype(torch::kLong));
  const int64_t ws_bytes = lvllm_skinny_gemm_argmax_workspace_bytes((int)M);
  auto ws = torch::empty({ws_bytes / 4}, x.options().dtype(torch::kFloat));
  check(lvllm_skinny_gemm_w8a8_ex(tokens.data_ptr(), x.data_ptr(), w_packed.data_ptr(), nullptr,
                                  x_scale.data_ptr<float>(), w_scale.data_ptr<float>(), (int)M, (int)N, (int)K,
                                  x.stride(0), dtype_code(x, "skinny_linear_w8a8_argmax"), 3, ws.data_ptr(), ws_bytes,
                                  current_stream(x)));
  return tokens;
}

torch::Tensor pack_weight(const torch::Tensor& w) {
  TORCH_CHECK(w.is_cuda() && w.dim() == 2 && w.is_contiguous(), "pack_weight: contiguous [N,K] GPU tensor");
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(w));
  auto out = torch::empty_like(w);
  check(lvllm_pack_weight(out.data_ptr(), w.data_ptr(), (int)w.size(0), (int)w.size(1),
                          dtype_code(w, "pack_weight"), current_stream(w)));
  return out;
}

int64_t get_device_attribute(int64_t attribute, int64_t device_id) {
  return lvllm_get_device_attribute(attribute, device_id);
}
int64_t get_max_shared_memory_per_block_device_attribute(int64_t device_id) {
  return lvllm_get_max_shared_memory_per_block_device_attribute(device_id);
}

}  // namespace

TORCH_LIBRARY_FRAGMENT(_C, ops) {
  // prepare_inputs advance_step (torch_bindings.cpp:75-77 of the reference, schema inferred there)
  ops.def("advance_step(int num_seqs, int num_queries, int block_size, Tensor! input_tokens, "
          "Tensor sampled_token_ids, Tensor! input_positions, Tensor! seq_lens, Tensor! slot_mapping, "
          "Tensor block_tables) -> ()");
  ops.impl("advance_step", torch::kCUDA, &advance_step);
}

TORCH_LIBRARY_FRAGMENT(_C_cache_ops, cache_ops) {
  // torch_bindings.cpp:261-264 of the reference
  cache_ops.def("convert_fp8(Tensor! dst_cache, Tensor src_cache, float scale, str kv_cache_dtype) -> ()");
  cache_ops.impl("convert_fp8", torch::kCUDA, &convert_fp8);

  cache_ops.def("swap_blocks(Tensor src, Tensor! dst, Tensor block_mapping) -> ()");
  cache_ops.impl("swap_blocks", torch::kCUDA, &swap_blocks);
  // a D2H swap dispatches on its CPU destination when src is listed first
  // only for CUDA; register CPU too so CPU->GPU and GPU->CPU both resolve
  cache_ops.impl("swap_blocks", torch::kCPU, &swap_blocks);

  cache_ops.def(
      "copy_blocks(Tensor[]! key_caches, Tensor[]! value_caches, Tensor "
      "block_mapping) -> ()");
  cache_ops.impl("copy_blocks", torch::kCUDA, &copy_blocks);

  cache_ops.def(
      "reshape_and_cache(Tensor key, Tensor value,"
      "                  Tensor! key_cache, Tensor! value_cache,"
      "                  Tensor slot_mapping,"
      "                  str kv_cache_dtype,"
      "                  float k_scale, float v_scale) -> ()");
  cache_ops.impl("reshape_and_cache", torch::kCUDA, &reshape_and_cache);

  cache_ops.def(
      "reshape_and_cache_flash(Tensor key, Tensor value,"
      "                        Tensor! key_cache,"
      "                        Tensor! value_cache,"
      "                        Tensor slot_mapping,"
      "                        str kv_cache_dtype,"
      "                        float k_scale, float v_scale) -> ()");
  cache_ops.impl("reshape_and_cache_flash", torch::kCUDA, &reshape_and_cache_flash);
}

TORCH_LIBRARY_FRAGMENT(_C_amd, amd) {
  amd.def("skinny_linear(Tensor x, Tensor w, Tensor? bias) -> Tensor");
  amd.impl("skinny_linear", torch::kCUDA, &skinny_linear);
  amd.def("skinny_linear_packed(Tensor x, Tensor w_packed, Tensor? bias, int N, int K) -> Tensor");
  amd.impl("skinny_linear_packed", torch::kCUDA, &skinny_linear_packed);
  amd.def("pack_weight(Tensor w) -> Tensor");
  amd.impl("pack_weight", torch::kCUDA, &pack_weight);
  amd.def("skinny_linear_packed_argmax(Tensor x, Tensor w_packed, int N, int K) -> Tensor");
  amd.impl("skinny_linear_packed_argmax", torch::kCUDA, &skinny_linear_packed_argmax);
  amd.def("skinny_linear_packed_clamped_unit(Tensor x, Tensor w_packed, int N, int K, float limit) -> Tensor");
  amd.impl("skinny_linear_packed_clamped_unit", torch::kCUDA, &skinny_linear_packed_clamped_unit);
  amd.def("clamped_unit(Tensor x, float limit) -> Tensor");
  amd.impl("clamped_unit", torch::kCUDA, &clamped_unit);
  amd.def("silu_unit(Tensor x) -> Tensor");
  amd.impl("silu_unit", torch::kCUDA, &silu_unit);
  amd.def("skinny_linear_packed_relu_squared(Tensor x, Tensor w_packed, int N, int K) -> Tensor");
  amd.impl("skinny_linear_packed_relu_squared", torch::kCUDA, &skinny_linear_packed_relu_squared);
  amd.def("stream_linear_packed(Tensor x, Tensor w_packed, Tensor? bias, int N, int K) -> Tensor");
  amd.impl("stream_linear_packed", torch::kCUDA, &stream_linear_packed);
  amd.def("skinny_linear_packed_swiglu(Tensor x, Tensor w_packed, Tensor? bias, int N, int K) -> Tensor");
  amd.impl("skinny_linear_packed_swiglu", torch::kCUDA, &skinny_linear_packed_swiglu);
  amd.def("skinny_linear_packed_partials(Tensor x, Tensor w_packed, int N, int K, bool swiglu) -> Tensor");
  amd.impl("skinny_linear_packed_partials", torch::kCUDA, &skinny_linear_packed_partials);
  amd.def("skinny_linear_w8a8(Tensor x, Tensor w_packed, Tensor w_scale, Tensor x_scale, int N, int K, "
          "Tensor? bias) -> Tensor");
  amd.impl("skinny_linear_w8a8", torch::kCUDA, &skinny_linear_w8a8);
  amd.def("skinny_linear_w8a8_swiglu(Tensor x, Tensor w_packed, Tensor w_scale, Tensor x_scale, int N, int K, "
          "Tensor? bias) -> Tensor");
  amd.impl("skinny_linear_w8a8_swiglu", torch::kCUDA, &skinny_linear_w8a8_swiglu);
  amd.def("skinny_linear_w8a8_argmax(Tensor x, Tensor w_packed, Tensor w_scale, Tensor x_scale, int N, int K) -> Tensor");
  amd.impl("skinny_linear_w8a8_argmax", torch::kCUDA, &skinny_linear_w8a8_argmax);
  amd.def("skinny_linear_w8a8_partials(Tensor x, Tensor w_packed, Tensor w_scale, Tensor x_scale, int N, int K) -> Tensor");
  amd.impl("skinny_linear_w8a8_partials", torch::kCUDA, &skinny_linear_w8a8_partials);
  amd.def("advance_step_logged(int block_size, Tensor! input_tokens, Tensor sampled_token_ids, "
          "Tensor! input_positions, Tensor! seq_lens, Tensor! slot_mapping, Tensor block_tables, "
          "Tensor! token_log) -> ()");
  amd.impl("advance_step_logged", torch::kCUDA, &advance_step_logged);
  amd.def("skinny_linear_w8a8_q(Tensor x_fp8, Tensor w_packed, Tensor w_scale, Tensor x_scale, int N, int K, "
          "Tensor? bias, ScalarType out_dtype) -> Tensor");
  amd.impl("skinny_linear_w8a8_q", torch::kCUDA, &skinny_linear_w8a8_q);
  amd.def("skinny_linear_w8a8_q_swiglu_fp8(Tensor x_fp8, Tensor w_packed, Tensor w_scale, Tensor x_scale, int N, int K, "
          "Tensor q_scale, ScalarType compute_dtype) -> Tensor");
  amd.impl("skinny_linear_w8a8_q_swiglu_fp8", torch::kCUDA, &skinny_linear_w8a8_q_swiglu_fp8);
  amd.def("skinny_linear_w8a8_q_partials(Tensor x_fp8, Tensor w_packed, Tensor w_scale, Tensor x_scale, int N, int K) "
          "-> Tensor");
  amd.impl("skinny_linear_w8a8_q_partials", torch::kCUDA, &skinny_linear_w8a8_q_partials);
  amd.def("sample_rows(Tensor! tokens_out, Tensor logits, Tensor? state_slot, Tensor(a!)? params, Tensor(b!)? counts, "
          "Tensor(c!)? scratch, Tensor(d!)? processed_out, bool update_state) -> ()");
  amd.impl("sample_rows", torch::kCUDA, &sample_rows);
  amd.def("sampler_init_row(Tensor! counts_row, Tensor prompt_tokens, Tensor output_tokens) -> ()");
  amd.impl("sampler_init_row", torch::kCUDA, &sampler_init_row);
  amd.def("set_tuning(str key, int value) -> ()", [](const std::string& key, int64_t value) {
    check(lvllm_set_tuning(key.c_str(), (int)value));
  });
  amd.def("get_tuning(str key) -> int", [](const std::string& key) {
    int v = 0;
    check(lvllm_get_tuning(key.c_str(), &v));
    return (int64_t)v;
  });
}

TORCH_LIBRARY_FRAGMENT(_C_cuda_utils, cuda_utils) {
  cuda_utils.def("get_device_attribute", &get_device_attribute);
  cuda_utils.def("get_max_shared_memory_per_block_device_attribute",
                 &get_max_shared_memory_per_block_device_attribute);
}

PyMODINIT_FUNC PyInit__C_base(void) {
  static struct PyModuleDef module = {PyModuleDef_HEAD_INIT, "_C_base", nullptr, 0, nullptr};
  return PyModule_Create(&module);
}
