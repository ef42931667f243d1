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
  const int32_t* tiles;   // [max_tiles + 1][2]: expert, first slot (expert < 0: none); last: tiles of all but the last expert, of all
  int experts, slots, rows, width, ff_max, max_tiles;
  int ff_first, ff_last;  // largest ffp of all experts but the last, the last one's
};

__device__ __forceinline__ float clamped_gate(float g, float u, float limit) {
  g = fminf(g, limit);
  u = fminf(fmaxf(u, -limit), limit);
  return g / (1.f + expf(-1.702f * g)) * (u + 1.f);
}

constexpr int kMaxExperts = 1024;

// The `top` largest of z[0 .. experts) (LDS; ties: the smaller index) by one wave, their softmax, and the shared expert.
// Any z gives indices in range.
__device__ __forceinline__ void choose_experts(float* z, int experts, int top, bool shared, int32_t* ids, float* weights) {
  const int lane = threadIdx.x & 63;
  float first = 0.f, sum = 0.f, mine = 0.f;
  for (int k = 0; k < top; ++k) {
    float best = -INFINITY;
    int at = kMaxExperts;
    for (int e = lane; e < experts; e += 64) {
      const float v = z[e];
      if (v > best || (at == kMaxExperts && v == v && v != -INFINITY)) { best = v; at = e; }
    }
#pragma unroll
    for (int m = 32; m >= 1; m >>= 1) {
      const float ob = __shfl_xor(best, m);
      const int oa = __shfl_xor(at, m);
      if (oa < kMaxExperts && (at == kMaxExperts || ob > best || (ob == best && oa < at))) { best = ob; at = oa; }
    }
    if (at >= kMaxExperts) {  // nothing comparable left: the first one not taken (marked by -inf) or, among NaNs, the k-th
      at = k;
      best = first;
    }
    if (k == 0) first = best;
    const float e = expf(best - first);
    sum += e;
    if (lane == k) mine = e;
    if (lane == 0) {
      ids[k] = at;
      z[at] = -INFINITY;
    }
    __builtin_amdgcn_wave_barrier();
    __threadfence_block();
  }
  if (lane < top) weights[lane] = mine / sum;
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
