// Mixture of experts for gfx950.  A token takes the `top` experts of the largest logits, weighted by the softmax over the chosen
// ones or each by its own sigmoid, times `scale`, and, as one more assignment, the shared expert, with a gate of its own or the
// weight 1.  With groups (equal runs of neighbouring experts) only the experts of the `keep` groups whose best logits are the
// largest can be chosen.  The step's assignments are grouped by expert: slot s of the grouped order belongs to row token[s]; expert
// e owns slots offsets[e] .. offsets[e + 1].
//
// Expert weights are two matrices per expert in one buffer:
//   up    [2 ffp, width]: 16 gate rows, 16 value rows, 16 gate rows, ... (ffp: the inner size, zero rows up to a multiple of 32)
//   down  [width, ffp]
// row-major or, where the matrix-core bodies run, packed as lvllm_pack_weight does.  The activation is
//   g = min(gate, limit), u = clamp(value, -limit, limit), a = g * sigmoid(1.702 g) * (u + 1)   (LVLLM_MOE_CLAMPED), or
//   a = gate * sigmoid(gate) * value                                                        (LVLLM_MOE_SILU)
// or, without gate rows (up [ffp, width]),
//   a = max(value, 0)^2                                                                     (LVLLM_MOE_RELU_SQUARED)
// where an assignment's weight may scale the expert's input, that is gate and value, instead of its output (slot_weight).
#pragma once
#include "common.h"

namespace lvllm {

// The products of an expert: up with gate rows, up without, down
enum { kMoeGated = 0, kMoePlain = 1, kMoeDown = 2 };

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
  const float* slot_weight;  // [slots] or null
  int act;                // LVLLM_MOE_CLAMPED, LVLLM_MOE_SILU or LVLLM_MOE_RELU_SQUARED
  int experts, slots, rows, width, ff_max, max_tiles;
  int ff_first, ff_last;  // largest ffp of all experts but the last, the last one's
};

// gate and value of a slot of expert e -> its activation
struct MoeActivation {
  float limit;
  bool silu;
  __device__ __forceinline__ MoeActivation(const MoeParams& p, int e) : limit(0.f), silu(p.act == LVLLM_MOE_SILU) {
    if (!silu && e >= 0) limit = p.limit[e];
  }
  __device__ __forceinline__ float operator()(float g, float u) const {
    return silu ? g / (1.f + expf(-g)) * u : clamped_unit_of(g, u, limit);
  }
};
__device__ __forceinline__ float slot_weight_of(const MoeParams& p, int slot) {
  return p.slot_weight != nullptr ? p.slot_weight[slot] : 1.f;
}

// How a token's assignments are found: experts and a last shared one (`gated`: weighted by its own logit's sigmoid)
struct MoeRouting {
  int experts, top, scoring;
  bool shared, gated;
  int groups, keep;  // groups <= 1: none
  float scale;
  __host__ __device__ __forceinline__ int logits() const { return experts + gated; }
  __host__ __device__ __forceinline__ int all() const { return experts + shared; }
  __host__ __device__ __forceinline__ int per_row() const { return top + shared; }
};

constexpr int kMaxExperts = 1024, kMaxGroups = 64;

// Logits of groups that are not among the `keep` best (ties: the earlier group) become -INFINITY; by one wave, a lane per group.
__device__ __forceinline__ void close_groups(float* z, const MoeRouting& r) {
  const int lane = threadIdx.x & 63, size = r.experts / r.groups;
  float best = -INFINITY;
  if (lane < r.groups)
    for (int e = lane * size; e < (lane + 1) * size; ++e) best = fmaxf(best, z[e]);
  int place = 0;
  for (int j = 0; j < r.groups; ++j) {
    const float o = __builtin_bit_cast(float, __builtin_amdgcn_readlane(__builtin_bit_cast(int, best), j));
    place += o > best || (o == best && j < lane);
  }
  const uint64_t open = __ballot(lane < r.groups && place < r.keep);
  for (int e = lane; e < r.experts; e += 64)
    if (!(open >> (e / size) & 1)) z[e] = -INFINITY;
  asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");  // (the wave's own next reads see it)
}

// The `top` largest of z[0 .. experts) (LDS; ties: the smaller index) by one wave, their weights, and the shared expert.  NaNs
// come last; any z gives distinct indices in range.
__device__ __forceinline__ void choose_experts(float* z, const MoeRouting& r, int32_t* ids, float* weights) {
  const int experts = r.experts, top = r.top;
  if (r.groups > 1) close_groups(z, r);
  const bool sigmoid = r.scoring == LVLLM_MOE_SIGMOID;
  const int lane = threadIdx.x & 63;
  auto value = [&](int e) {
    const float v = z[e];
    return v == v ? v : -INFINITY;
  };
  auto weight_of = [&](float v, float mx) {
    return v == -INFINITY ? 1e-30f : sigmoid ? 1.f / (1.f + expf(-v)) : expf(v - mx);
  };
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
    const float sum = sigmoid ? 1.f : wave_sum(w);
    if (chosen) {
      ids[place] = lane;
      weights[place] = w / sum * r.scale;
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
          weights[k] = (sigmoid ? w : w / sum) * r.scale;
        }
      }
    }
  }
  if (r.shared && lane == 0) {
    ids[top] = experts;
    weights[top] = r.gated ? 1.f / (1.f + expf(-z[experts])) : 1.f;
  }
}

// Where the grouped assignments go: offsets [experts + 1], token and slot [assignments], tiles of `tile` slots, and (null: not
// kept) the assignments' weights in the order of the slots.  count [experts], zeroed: only for rows that count their own
// assignments (moe_count_assignments).
struct MoeGroups {
  int32_t *offsets, *token, *slot, *tiles, *count;
  int tile, max_tiles;
  const float* weights;  // [rows, per row]
  float* slot_weight;    // [assignments] or null
};
__device__ __forceinline__ void moe_place(const MoeGroups& out, int i, int per_row, int s) {
  out.slot[i] = s;
  out.token[s] = i / per_row;
  if (out.slot_weight != nullptr) out.slot_weight[s] = out.weights[i];
}

// Running sums of the experts' slots and tiles, 64 experts a turn, by the first wave; count, first [experts + 1] and tile0
// [experts + 1] in LDS.
__device__ __forceinline__ void moe_running_sums(const int* count, int* first, int* tile0, int experts, int tile) {
  if (threadIdx.x >= 64) return;
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

// offsets and tiles, by the whole workgroup
__device__ __forceinline__ void moe_write_tiles(const int* first, const int* tile0, int experts, const MoeGroups& out) {
  int32_t* tiles = out.tiles;
  for (int e = threadIdx.x; e <= experts; e += blockDim.x) out.offsets[e] = first[e];
  for (int e = threadIdx.x; e < experts; e += blockDim.x)
    for (int t = tile0[e]; t < tile0[e + 1] && t < out.max_tiles; ++t) {
      tiles[4 * t] = e;
      tiles[4 * t + 1] = first[e] + (t - tile0[e]) * out.tile;
      tiles[4 * t + 2] = tile0[e];
      tiles[4 * t + 3] = tile0[e + 1] - tile0[e];
    }
  for (int t = tile0[experts] + threadIdx.x; t < out.max_tiles; t += blockDim.x) tiles[4 * t] = -1;
  if (threadIdx.x == 0) {
    tiles[4 * out.max_tiles] = min(tile0[experts - 1], out.max_tiles);
    tiles[4 * out.max_tiles + 1] = min(tile0[experts], out.max_tiles);
  }
}

// Everything of `total` assignments, by one workgroup of 1024.  `shared`: the last assignment of every row is the last
// expert's, in row order.
__device__ __forceinline__ void group_assignments(const int32_t* ids, const int total, const int per_row, const int experts,
                                                  const int shared, const MoeGroups& out) {
  __shared__ int count[kMaxExperts + 1], first[kMaxExperts + 2], tile0[kMaxExperts + 2];
  for (int e = threadIdx.x; e < experts; e += 1024) count[e] = shared && e == experts - 1 ? total / per_row : 0;
  __syncthreads();
  for (int i = threadIdx.x; i < total; i += 1024) {
    const int e = min(max(ids[i], 0), experts - 1);
    out.slot[i] = shared && e == experts - 1 ? i / per_row : atomicAdd(&count[e], 1);
  }
  __syncthreads();
  moe_running_sums(count, first, tile0, experts, out.tile);
  __syncthreads();
  for (int i = threadIdx.x; i < total; i += 1024) {
    moe_place(out, i, per_row, first[min(max(ids[i], 0), experts - 1)] + out.slot[i]);
  }
  moe_write_tiles(first, tile0, experts, out);
}

// Many rows: a workgroup that has chosen for rows row0 .. row0 + n - 1 counts their assignments -- in LDS (`local`, experts
// long), then once per expert in memory -- and leaves every assignment's rank among its expert's in `slot`; the running sums
// and the final slots are a launch each (launch_moe_group).
__device__ __forceinline__ void moe_count_assignments(const int32_t* ids, int row0, int n, int per_row, int experts, int shared,
                                                      int* local, const MoeGroups& out) {
  for (int e = threadIdx.x; e < experts; e += blockDim.x) local[e] = 0;
  __syncthreads();
  const int total = n * per_row;
  for (int i = threadIdx.x; i < total; i += blockDim.x) {
    const int at = row0 * per_row + i, e = min(max(ids[at], 0), experts - 1);
    const bool last = shared && e == experts - 1;
    out.slot[at] = last ? row0 + i / per_row : atomicAdd(&local[e], 1);
  }
  __syncthreads();
  for (int e = threadIdx.x; e < experts; e += blockDim.x)
    if (local[e] > 0) local[e] = atomicAdd(&out.count[e], local[e]);
  __syncthreads();
  for (int i = threadIdx.x; i < total; i += blockDim.x) {
    const int at = row0 * per_row + i, e = min(max(ids[at], 0), experts - 1);
    if (!(shared && e == experts - 1)) out.slot[at] += local[e];
  }
}

// slots of a tile: of the matrix-core body for prompts, and of those for few rows and for sizes without one
constexpr int kMoeTile = 128, kMoeSmallTile = 16, kMoeFewRows = 64;
inline int moe_tile(bool packed, int rows) { return packed && rows > kMoeFewRows ? kMoeTile : kMoeSmallTile; }

bool moe_takes_mfma(int width, int dtype);
int launch_moe_mfma(const MoeParams& p, int product, hipStream_t s);
// `counted`: the rows have counted their assignments
int launch_moe_group(const int32_t* ids, int total, int per_row, int experts, int shared, bool counted, const MoeGroups& groups,
                     hipStream_t s);
int64_t moe_route_mfma_workspace(const MoeRouting& r, int rows, int width);
int launch_moe_route_mfma(int32_t* ids, float* weights, const void* h, const void* w, const float* bias, const MoeRouting& r,
                          int rows, int width, const MoeGroups& groups, float* workspace, hipStream_t s);

}  // namespace lvllm
