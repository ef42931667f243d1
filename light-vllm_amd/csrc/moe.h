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

// The `top` largest of z[0 .. experts) (LDS; ties: the smaller index) by one wave, their softmax, and the shared expert.  NaNs
// come last; any z gives distinct indices in range.
__device__ __forceinline__ void choose_experts(const float* z, int experts, int top, bool shared, int32_t* ids, float* weights) {
  const int lane = threadIdx.x & 63;
  auto value = [&](int e) {
    const float v = z[e];
    return v == v ? v : -INFINITY;
  };
  auto weight_of = [](float v, float mx) { return v == -INFINITY ? 1e-30f : expf(v - mx); };
  if (experts <= 64) {  // a logit's place is the number of logits ahead of it
    const float v = lane < experts ? value(lane) : -INFINITY;
    int place = 0;
    for (int j = 0; j < experts; ++j) {
      const float o = __builtin_bit_cast(float, __builtin_amdgcn_readlane(__builtin_bit_cast(int, v), j));
      place += o > v || (o == v && j < lane);
    }
    const bool chosen = lane < experts && place < top;
    const float mx = wave_max(v);  // (by all lanes)
    const float w = chosen ? weight_of(v, mx) : 0.f;
    const float sum = wave_sum(w);
    if (chosen) {
      ids[place] = lane;
      weights[place] = w / sum;
    }
  } else {  // one after the other; `taken`: which of this lane's logits are gone
    uint32_t taken = 0;
    float first = 0.f, sum = 0.f;
    for (int pass = 0; pass < 2; ++pass) {  // the chosen ones' sum, then their weights
      taken = 0;
      for (int k = 0; k < top; ++k) {
        float best = -INFINITY;
        int at = kMaxExperts;
        for (int e = lane, i = 0; e < experts; e += 64, ++i) {
          const float v = value(e);
          if (!(taken >> i & 1) && (at == kMaxExperts || v > best)) { best = v; at = e; }
        }
#pragma unroll
        for (int m = 32; m >= 1; m >>= 1) {
          const float ob = __shfl_xor(best, m);
          const int oa = __shfl_xor(at, m);
          if (oa < kMaxExperts && (at == kMaxExperts || ob > best || (ob == best && oa < at))) { best = ob; at = oa; }
        }
        if ((at & 63) == lane) taken |= 1u << (at >> 6);
        if (k == 0) first = best;
        const float w = weight_of(best, first);
        if (pass == 0) {
          sum += w;
        } else if (lane == 0) {
          ids[k] = at;
          weights[k] = w / sum;
        }
      }
    }
  }
  if (shared && lane == 0) {
    ids[top] = experts;
    weights[top] = 1.f / (1.f + expf(-z[experts]));
  }
}

// Where the grouped assignments go: offsets [experts + 1], token and slot [assignments], tiles of `tile` slots.
struct MoeGroups {
  int32_t *offsets, *token, *slot, *tiles;
  int tile, max_tiles;
};

// Counts, offsets, slots and tiles of `total` assignments, by one workgroup of 1024.  `shared`: the last assignment of every
// row is the last expert's, in row order.
__device__ __forceinline__ void group_assignments(const int32_t* ids, const int total, const int per_row, const int experts,
                                                  const int shared, const MoeGroups& out) {
  int32_t *offsets = out.offsets, *token = out.token, *slot = out.slot, *tiles = out.tiles;
  const int tile = out.tile, max_tiles = out.max_tiles;
  __shared__ int count[kMaxExperts + 1], first[kMaxExperts + 2], tile0[kMaxExperts + 2];
  for (int e = threadIdx.x; e < experts; e += 1024) count[e] = shared && e == experts - 1 ? total / per_row : 0;
  __syncthreads();
  constexpr int B = 8;  // loads in flight
  for (int i0 = threadIdx.x; i0 < total; i0 += 1024 * B) {
    int e[B];
#pragma unroll
    for (int j = 0; j < B; ++j) e[j] = i0 + 1024 * j < total ? min(max(ids[i0 + 1024 * j], 0), experts - 1) : -1;
#pragma unroll
    for (int j = 0; j < B; ++j)
      if (e[j] >= 0) e[j] = shared && e[j] == experts - 1 ? (i0 + 1024 * j) / per_row : atomicAdd(&count[e[j]], 1);
#pragma unroll
    for (int j = 0; j < B; ++j)
      if (i0 + 1024 * j < total) slot[i0 + 1024 * j] = e[j];
  }
  __syncthreads();
  if (threadIdx.x < 64) {  // running sums, 64 experts a turn
    int base = 0, tbase = 0;
    for (int e0 = 0; e0 < experts; e0 += 64) {
      const int e = e0 + threadIdx.x;
      const int c = e < experts ? count[e] : 0, t = (c + tile - 1) / tile;
      int s = c, ts = t;
#pragma unroll
      for (int d = 1; d < 64; d <<= 1) {
        const int a = __shfl_up(s, d), b = __shfl_up(ts, d);
        if ((int)threadIdx.x >= d) { s += a; ts += b; }
      }
      if (e < experts) { first[e] = base + s - c; tile0[e] = tbase + ts - t; }
      base += __shfl(s, 63);
      tbase += __shfl(ts, 63);
    }
    if (threadIdx.x == 0) { first[experts] = base; tile0[experts] = tbase; }
  }
  __syncthreads();
  for (int e = threadIdx.x; e <= experts; e += 1024) offsets[e] = first[e];
  for (int i0 = threadIdx.x; i0 < total; i0 += 1024 * B) {
    int e[B], s[B];
#pragma unroll
    for (int j = 0; j < B; ++j) {
      const int i = min(i0 + 1024 * j, total - 1);
      e[j] = min(max(ids[i], 0), experts - 1);
      s[j] = slot[i];
    }
#pragma unroll
    for (int j = 0; j < B; ++j) {
      const int i = i0 + 1024 * j;
      if (i >= total) break;
      slot[i] = first[e[j]] + s[j];
      token[first[e[j]] + s[j]] = i / per_row;
    }
  }
  for (int e = threadIdx.x; e < experts; e += 1024)
    for (int t = tile0[e]; t < tile0[e + 1] && t < max_tiles; ++t) {
      tiles[4 * t] = e;
      tiles[4 * t + 1] = first[e] + (t - tile0[e]) * tile;
      tiles[4 * t + 2] = tile0[e];
      tiles[4 * t + 3] = tile0[e + 1] - tile0[e];
    }
  for (int t = tile0[experts] + threadIdx.x; t < max_tiles; t += 1024) tiles[4 * t] = -1;
  if (threadIdx.x == 0) {
    tiles[4 * max_tiles] = min(tile0[experts - 1], max_tiles);
    tiles[4 * max_tiles + 1] = min(tile0[experts], max_tiles);
  }
}

// slots of a tile: of the matrix-core body for prompts, and of those for few rows and for sizes without one
constexpr int kMoeTile = 128, kMoeSmallTile = 16, kMoeFewRows = 64;
inline int moe_tile(bool packed, int rows) { return packed && rows > kMoeFewRows ? kMoeTile : kMoeSmallTile; }

bool moe_takes_mfma(int width, int dtype);
int launch_moe_mfma(const MoeParams& p, bool up, hipStream_t s);
int launch_moe_group(const int32_t* ids, int total, int per_row, int experts, int shared, const MoeGroups& groups, hipStream_t s);
int64_t moe_route_mfma_workspace(int experts, int shared, int rows, int width);
int launch_moe_route_mfma(int32_t* ids, float* weights, const void* h, const void* w, const float* bias, int experts, int shared,
                          int top, int rows, int width, const MoeGroups& groups, float* workspace, hipStream_t s);

}  // namespace lvllm
