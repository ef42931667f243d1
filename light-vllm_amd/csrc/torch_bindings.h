// Helpers shared by the torch op registrations (torch_bindings*.cpp): dtype codes, argument
// checks, the current stream, the C-ABI's error string as an exception.  Host-only C++.
#pragma once
#include <Python.h>
#include <ATen/hip/impl/HIPGuardImplMasqueradingAsCUDA.h>
#include <ATen/hip/impl/HIPStreamMasqueradingAsCUDA.h>
#include <torch/all.h>
#include <torch/library.h>

#include <optional>
#include <string>
#include <vector>

#include "lvllm_hip.h"

namespace {

[[maybe_unused]] int dtype_code(const torch::Tensor& t, const char* what) {
  switch (t.scalar_type()) {
    case at::ScalarType::Float: return LVLLM_F32;
    case at::ScalarType::Half: return LVLLM_F16;
    case at::ScalarType::BFloat16: return LVLLM_BF16;
    default: TORCH_CHECK(false, what, ": unsupported dtype ", t.scalar_type());
  }
}

// kv_cache_dtype strings: csrc/quantization/fp8/amd/quant_utils.cuh:547-573
[[maybe_unused]] int kv_dtype_code(const std::string& s) {
  if (s == "auto") return LVLLM_KV_AUTO;
  if (s == "fp8" || s == "fp8_e4m3") return LVLLM_KV_FP8_E4M3;
  TORCH_CHECK(false, "Unsupported data type of kv cache: ", s);
}

// "auto": the cache holds the query's element type; "fp8": one byte per element
[[maybe_unused]] void check_cache_dtype(const torch::Tensor& cache, const torch::Tensor& like, int kv_code, const char* op) {
  if (kv_code == LVLLM_KV_AUTO) {
    TORCH_CHECK(cache.scalar_type() == like.scalar_type(), op, ": kv_cache_dtype 'auto' needs a cache of dtype ",
                like.scalar_type(), ", got ", cache.scalar_type());
  } else {
    TORCH_CHECK(cache.element_size() == 1, op, ": kv_cache_dtype 'fp8' needs a one-byte cache dtype, got ",
                cache.scalar_type());
  }
}

// Bytes the kernels may touch behind key_cache.data_ptr() / value_cache.data_ptr() (the smaller of the two):
// the C-ABI clamps block numbers / skips slots beyond it instead of following them out of the allocation.
[[maybe_unused]] int64_t cache_extent_bytes(const torch::Tensor& key_cache, const torch::Tensor& value_cache) {
  auto bytes = [](const torch::Tensor& t) {
    return t.dim() == 0 ? (int64_t)0 : t.size(0) * t.stride(0) * (int64_t)t.element_size();
  };
  const int64_t k = bytes(key_cache), v = bytes(value_cache);
  return k < v ? k : v;
}

// A paged cache as the kernels address it: every block dense ([KVH, D/x, BS, x] or [KVH, D, BS] contiguous), blocks
// stride(0) elements apart -- the dense product, or more when the allocation pads its blocks.
[[maybe_unused]] bool blocks_are_dense(const torch::Tensor& t) {
  if (t.dim() < 2) return t.is_contiguous();
  int64_t expect = 1;
  for (int64_t d = t.dim() - 1; d >= 1; --d) {
    if (t.size(d) != 1 && t.stride(d) != expect) return false;
    expect *= t.size(d);
  }
  return t.stride(0) >= expect;
}

[[maybe_unused]] void* current_stream(const torch::Tensor& t) {
  return (void*)c10::hip::getCurrentHIPStreamMasqueradingAsCUDA(t.device().index()).stream();
}

[[maybe_unused]] void check(int rc) { TORCH_CHECK(rc == 0, lvllm_last_error()); }

#define LV_CHECK_DEVICE(t) TORCH_CHECK((t).is_cuda(), #t " must be a GPU tensor")

// ---- the W8A8 decode step with activations quantised ONCE, by their producer (include/lvllm_hip.h: *_quant entries,
// lvllm_skinny_gemm_w8a8_q): every op below is bit-identical to the op it stands for followed by / preceded by
// static_scaled_fp8_quant
[[maybe_unused]] void check_q_scale(const torch::Tensor& s, const char* op) {
  TORCH_CHECK(s.is_cuda() && s.scalar_type() == at::kFloat && s.numel() == 1, op, ": one float32 scale on the device");
}

// ---- decoders of listed layers (include/lvllm_hip.h) ----
// a step's layout: [num_seqs + 1] / [num_seqs] int32 on the device
[[maybe_unused]] void check_layout(const torch::Tensor& query_start_loc, const torch::Tensor& seq_lens, const char* op) {
  TORCH_CHECK(query_start_loc.is_cuda() && seq_lens.is_cuda() && query_start_loc.scalar_type() == at::kInt &&
                  seq_lens.scalar_type() == at::kInt && query_start_loc.is_contiguous() && seq_lens.is_contiguous() &&
                  query_start_loc.numel() == seq_lens.numel() + 1,
              op, ": query_start_loc int32 [num_seqs + 1] and seq_lens int32 [num_seqs] on the device");
}
[[maybe_unused]] void check_f32(const torch::Tensor& t, int64_t numel, const char* op, const char* what) {
  TORCH_CHECK(t.is_cuda() && t.scalar_type() == at::kFloat && t.is_contiguous() && t.numel() == numel, op, ": ", what,
              " must be ", numel, " contiguous float32 elements on the device");
}
// [slots, ...] float32, dense behind dim 0
[[maybe_unused]] void check_state(const torch::Tensor& t, const torch::Tensor& slots, int64_t numel, int64_t num_seqs, const char* op) {
  TORCH_CHECK(t.is_cuda() && t.scalar_type() == at::kFloat && t.dim() >= 2 && blocks_are_dense(t) &&
                  t.numel() == t.size(0) * numel,
              op, ": state must be float32 [slots, ", numel, " elements], dense behind its first dimension");
  TORCH_CHECK(slots.is_cuda() && slots.scalar_type() == at::kInt && slots.is_contiguous() && slots.numel() >= num_seqs, op,
              ": state_slots int32 [num_seqs] on the device");
}
// a projection result as an addend: [rows, width] of the compute dtype, or fp32 slabs [s, rows, width]
struct Addend {
  const void* y = nullptr;
  const float* partials = nullptr;
  int num = 0;
};
[[maybe_unused]] Addend addend_of(const std::optional<torch::Tensor>& y, const torch::Tensor& x, at::ScalarType dtype, const char* op) {
  Addend a;
  if (!y) return a;
  TORCH_CHECK(y->is_cuda() && y->is_contiguous(), op, ": y must be contiguous on the device");
  if (y->dim() == 3) {
    TORCH_CHECK(y->scalar_type() == at::kFloat && y->size(1) == x.size(0) && y->size(2) == x.size(1), op,
                ": partials must be float32 [s, rows, width]");
    a.partials = y->data_ptr<float>();
    a.num = (int)y->size(0);
  } else {
    TORCH_CHECK(y->scalar_type() == dtype && y->sizes() == x.sizes(), op, ": y must be [rows, width] of the compute dtype");
    a.y = y->data_ptr();
  }
  return a;
}
[[maybe_unused]] void check_residual(const torch::Tensor& x, const char* op) {
  TORCH_CHECK(x.is_cuda() && x.dim() == 2 && x.is_contiguous() && x.scalar_type() == at::kFloat, op,
              ": the residual must be contiguous float32 [rows, width]");
}

// caches as lvllm_qk_norm_cache describes them; returns (kpad, vpad, block_size)
[[maybe_unused]] std::tuple<int64_t, int64_t, int64_t> head_cache_dims(const torch::Tensor& kc, const torch::Tensor& vc, int64_t kv_heads,
                                                      at::ScalarType dtype, const char* op) {
  TORCH_CHECK(kc.is_cuda() && vc.is_cuda() && kc.dim() == 5 && vc.dim() == 4 && kc.size(0) == vc.size(0) &&
                  kc.size(1) == kv_heads && vc.size(1) == kv_heads && kc.size(3) == vc.size(3) &&
                  kc.scalar_type() == dtype && vc.scalar_type() == dtype && kc.size(4) * kc.element_size() == 16 &&
                  blocks_are_dense(kc) && blocks_are_dense(vc),
              op, ": key_cache [blocks, kv_heads, kpad/x, block_size, x] and value_cache [blocks, kv_heads, vpad, block_size]");
  return {kc.size(2) * kc.size(4), vc.size(2), vc.size(3)};
}

// rotary positions, rows of projections, integer tables, block tables
[[maybe_unused]] void check_rot(const torch::Tensor& positions, const torch::Tensor& turns, int64_t rows, const char* op) {
  TORCH_CHECK(positions.is_cuda() && positions.scalar_type() == at::kLong && positions.is_contiguous() &&
                  positions.numel() >= rows && turns.is_cuda() && turns.scalar_type() == at::kDouble &&
                  turns.is_contiguous(),
              op, ": positions int64 [rows] and turns float64 [rot_dims / 2] on the device");
}
[[maybe_unused]] void check_rows2d(const torch::Tensor& t, int64_t rows, int64_t cols, at::ScalarType dtype, const char* op, const char* what) {
  TORCH_CHECK(t.is_cuda() && t.dim() == 2 && t.size(0) == rows && t.size(1) == cols && t.stride(1) == 1 &&
                  t.scalar_type() == dtype,
              op, ": ", what, " must be [", rows, ", ", cols, "] rows of the compute dtype");
}
[[maybe_unused]] void check_i32(const torch::Tensor& t, int64_t least, const char* op, const char* what) {
  TORCH_CHECK(t.is_cuda() && t.scalar_type() == at::kInt && t.is_contiguous() && t.numel() >= least, op, ": ", what,
              " must be ", least, " or more contiguous int32 elements on the device");
}
[[maybe_unused]] void check_tables(const torch::Tensor& block_tables, int64_t num_seqs, const char* op) {
  TORCH_CHECK(block_tables.is_cuda() && block_tables.dim() == 2 && block_tables.scalar_type() == at::kInt &&
                  block_tables.is_contiguous() && block_tables.size(0) >= num_seqs,
              op, ": block_tables int32 [num_seqs, blocks]");
}
[[maybe_unused]] void check_slots(const torch::Tensor& slot_mapping, int64_t rows, const char* op) {
  TORCH_CHECK(slot_mapping.is_cuda() && slot_mapping.scalar_type() == at::kLong && slot_mapping.is_contiguous() &&
                  slot_mapping.numel() >= rows,
              op, ": slot_mapping int64 [rows]");
}

}  // namespace
