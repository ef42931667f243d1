// Mixture of experts for gfx950.  A token takes its `top` experts (softmax over the chosen logits) and, as one more
// assignment, the shared expert with a gate of its own.  The step's assignments are grouped by expert: slot s of the grouped
// order belongs to row token[s]; expert e owns slots offsets[e] .. offsets[e + 1].
//
// Expert weights are two matrices per expert in one buffer:
//   up    [2 ffp, width]: 16 gate rows, 16 value rows, 16 gate rows, ... (ffp: the inner size, zero rows up to a multiple of 32)
//   down  [width, ffp]
// row-major or, where the matrix-core bodies run, packed as lvllm_pack_weight does.  The activation is
//   g = min(gate, limit), u = clamp(value, -limit, limit), a = g * sigmoid(1.702 g) * (u + 1).
#pragma once
#include "common.h"

namespace lvllm {

struct MoeParams {
  void* out;              // up: a [slots, ff_max]; down: y [slots, width]
  const void *x, *w;      // up: x [rows, width]; down: x = a
  const int64_t* w_offset;  // [experts] elements from w
  const int32_t *ff;      // [experts] ffp
  const float* limit;     // [experts]
  const int32_t *offsets, *token;
  const int32_t* tiles;   // [max_tiles][2]: expert, first slot (expert < 0: none)
  int experts, slots, rows, width, ff_max, max_tiles;
};

__device__ __forceinline__ float clamped_gate(float g, float u, float limit) {
  g = fminf(g, limit);
  u = fminf(fmaxf(u, -limit), limit);
  return g / (1.f + expf(-1.702f * g)) * (u + 1.f);
}

constexpr int kMoeTile = 128;       // slots of a tile of the matrix-core body
constexpr int kMoeSimpleTile = 16;

bool moe_takes_mfma(int width, int dtype);
int launch_moe_mfma(const MoeParams& p, bool up, hipStream_t s);

}  // namespace lvllm
