// torch op registrations of the moe library: routers and grouped products of mixtures of experts.
#include "torch_bindings.h"

namespace {

// (ids, weights, offsets, token, slots, tiles, slot_weight); w has a row per expert and, `gated`, one for the shared expert
std::tuple<torch::Tensor, torch::Tensor, torch::Tensor, torch::Tensor, torch::Tensor, torch::Tensor, torch::Tensor> moe_route(
    const torch::Tensor& h, const torch::Tensor& w, const std::optional<torch::Tensor>& bias, int64_t top, bool shared,
    bool packed, int64_t experts, bool gated, int64_t scoring, bool by_slot, int64_t groups, int64_t keep, double scale) {
  const char* op = "moe_route";
  LV_CHECK_DEVICE(h);
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(h));
  TORCH_CHECK(bias.has_value() || experts > 0, op, ": the number of experts comes with the bias or by itself");
  if (experts <= 0) experts = bias->numel();
  const int64_t rows = h.size(0), width = h.size(1), logits = experts + (shared && gated);
  TORCH_CHECK(h.dim() == 2 && h.is_contiguous() && w.is_cuda() && w.dim() == 2 && w.is_contiguous() && w.size(1) == width &&
                  w.scalar_type() == h.scalar_type() && w.size(0) == (packed ? (logits + 15) / 16 * 16 : logits),
              op, ": h [rows, width], w [logits, width], packed: rows up to a multiple of 16");
  if (bias) check_f32(*bias, experts, op, "bias");
  const lvllm_moe_routing routing{(int)experts, (int)top, (int)scoring,
                                  !shared ? LVLLM_MOE_NO_SHARED : gated ? LVLLM_MOE_GATED_SHARED : LVLLM_MOE_PLAIN_SHARED,
                                  (int)groups, (int)keep, (float)scale};
  const auto ints = h.options().dtype(at::kInt), floats = h.options().dtype(at::kFloat);
  const int64_t n = top + shared, total = rows * n, tile = lvllm_moe_tile(packed, (int)rows);
  const int64_t max_tiles = std::max<int64_t>(1, std::min(total, total / tile + experts + shared));
  auto ids = torch::empty({rows, n}, ints), slot = torch::empty({rows, n}, ints), token = torch::empty({total}, ints);
  auto offsets = torch::empty({experts + shared + 1}, ints), tiles = torch::empty({max_tiles + 1, 4}, ints);
  auto weights = torch::empty({rows, n}, floats), slot_weight = torch::empty({by_slot ? total : 0}, floats);
  const int64_t need = lvllm_moe_route_workspace_bytes(&routing, (int)rows, (int)width, packed);
  auto ws = torch::empty({need}, h.options().dtype(at::kByte));
  check(lvllm_moe_route(ids.data_ptr<int>(), weights.data_ptr<float>(), offsets.data_ptr<int>(), token.data_ptr<int>(),
                        slot.data_ptr<int>(), by_slot ? slot_weight.data_ptr<float>() : nullptr, tiles.data_ptr<int>(),
                        (int)max_tiles, h.data_ptr(), w.data_ptr(), bias ? bias->data_ptr<float>() : nullptr, &routing,
                        (int)rows, (int)width, packed, ws.data_ptr(), need, dtype_code(h, op), current_stream(h)));
  return {ids, weights, offsets, token, slot, tiles, slot_weight};
}

torch::Tensor moe_experts(const torch::Tensor& x, const torch::Tensor& w, const torch::Tensor& w_offset,
                          const torch::Tensor& ff, const std::optional<torch::Tensor>& limit, const torch::Tensor& offsets,
                          const torch::Tensor& token, const torch::Tensor& tiles, int64_t rows, int64_t width, int64_t ff_max,
                          int64_t ff_first, int64_t ff_last, bool up, bool packed,
                          const std::optional<torch::Tensor>& slot_weight, int64_t act) {
  const char* op = "moe_experts";
  LV_CHECK_DEVICE(x);
  const c10::hip::OptionalHIPGuardMasqueradingAsCUDA guard(device_of(x));
  const int64_t experts = ff.numel(), slots = token.numel();
  TORCH_CHECK(x.dim() == 2 && x.is_contiguous() && x.size(0) == (up ? rows : slots) && x.size(1) == (up ? width : ff_max), op,
              ": x must be [rows, width] going up, [slots, ff_max] going down");
  TORCH_CHECK(w.is_cuda() && w.is_contiguous() && w.scalar_type() == x.scalar_type() && w_offset.is_cuda() &&
                  w_offset.scalar_type() == at::kLong && w_offset.numel() == experts,
              op, ": one weight buffer and int64 offsets [experts]");
  check_i32(ff, experts, op, "ff");
  if (limit) check_f32(*limit, experts, op, "limit");
  if (slot_weight) check_f32(*slot_weight, slots, op, "slot_weight");
  check_i32(offsets, experts + 1, op, "offsets");
  check_i32(token, slots, op, "token");
  check_i32(tiles, 8, op, "tiles");
  auto out = torch::empty({slots, up ? ff_max : width}, x.options());
  check(lvllm_moe_experts(out.data_ptr(), x.data_ptr(), w.data_ptr(), w_offset.data_ptr<int64_t>(), ff.data_ptr<int>(),
                          limit ? limit->data_ptr<float>() : nullptr, slot_weight ? slot_weight->data_ptr<float>() : nullptr,
                          (int)act, offsets.data_ptr<int>(), token.data_ptr<int>(), tiles.data_ptr<int>(), (int)experts,
                          (int)slots, (int)rows, (int)width, (int)ff_max, (int)ff_first, (int)ff_last, (int)tiles.size(0) - 1,
                          up, packed, dtype_code(x, op), current_stream(x)));
  return out;
}

}  // namespace

TORCH_LIBRARY_FRAGMENT(_C_amd, moe) {
  moe.def("moe_route(Tensor h, Tensor w, Tensor? bias, int top, bool shared, bool packed, int experts=0, bool gated=True, "
          "int scoring=0, bool by_slot=False, int groups=1, int keep=1, float scale=1.) -> (Tensor, Tensor, Tensor, Tensor, Tensor, Tensor, Tensor)");
  moe.impl("moe_route", torch::kCUDA, &moe_route);
  moe.def("moe_experts(Tensor x, Tensor w, Tensor w_offset, Tensor ff, Tensor? limit, Tensor offsets, Tensor token, "
          "Tensor tiles, int rows, int width, int ff_max, int ff_first, int ff_last, bool up, bool packed, "
          "Tensor? slot_weight=None, int act=0) -> Tensor");
  moe.impl("moe_experts", torch::kCUDA, &moe_experts);
}

PyMODINIT_FUNC PyInit__C_moe(void) {
  static struct PyModuleDef module = {PyModuleDef_HEAD_INIT, "_C_moe", nullptr, 0, nullptr};
  return PyModule_Create(&module);
}
