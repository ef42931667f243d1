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
  // [max_tiles + 1][4]: expert (< 0: none), first slot, the expert's first tile and its number of tiles; the last entry: tiles
  // of all experts but the last one, tiles of all
  const int32_t* tiles;
  int experts, slots, rows, width, ff_max, max_tiles;
  int ff_first, ff_last;  // largest ffp of all experts but the last, the last one's
};

__device__ __forceinline__ float clamped_gate(float g, float u, float limit) {
  g = fminf(g, limit);
  u = fminf(fmaxf(u, -limit), limit);
  return g / (1.f + expf(-1.702f * g)) * (u + 1.f);
}

constexpr int kMaxExperts = 1024;

// The `top` largest of z[0 .. experts) (LDS; ties: the smaller index) by one wave, their softmax, and the shared expert.  Every
// logit's place is the number of logits ahead of it; NaNs come last, so that any z gives distinct indices in range.
__device__ __forceinline__ void choose_experts(const float* z, int experts, int top, bool shared, int32_t* ids, float* weights) {
  const int lane = threadIdx.x & 63;
  auto value = [&](int e) { return z[e] == z[e] ? z[e] : -INFINITY; };
  float mx = -INFINITY;
  for (int e = lane; e < experts; e += 64) mx = fmaxf(mx, value(e));
  mx = wave_max(mx);
  if (mx == -INFINITY) mx = 0.f;  // (nothing to compare)
  float sum = 0.f;
  for (int pass = 0; pass < 2; ++pass) {  // the chosen ones' sum, then their weights
    for (int e = lane; e < experts; e += 64) {
      const float v = value(e);
      int place = 0;
#pragma unroll 8
      for (int j = 0; j < experts; ++j) {
        const float o = value(j);
        place += o > v || (o == v && j < e);
      }
      if (place >= top) continue;
      const float w = v == -INFINITY ? 1e-30f : expf(v - mx);
      if (pass == 0) {
        sum += w;
      } else {
        ids[place] = e;
        weights[place] = w / sum;
      }
    }
    if (pass == 0) sum = wave_sum(sum);
  }
  if (shared && lane == 0) {
    ids[top] = experts;
    weights[top] = 1.f / (1.f + expf(-z[experts]));
  }
}

constexpr int kMoeTile = 128;       // slots of a tile of the matrix-core body
constexpr int kMoeSimpleTile = 16;

bool moe_takes_mfma(int width, int dtype);
int launch_moe_mfma(const MoeParams& p, bool up, hipStream_t s);
int launch_moe_route_mfma(int32_t* ids, float* weights, const void* h, const void* w, const float* bias, int experts, int shared,
                          int top, int rows, int width, hipStream_t s);

}  // namespace lvllm
