// Mixture of experts: the router, the grouping of a step's assignments, and the plain products (moe.h; the matrix-core
// bodies are in moe_mfma.hip).
#include "moe.h"

namespace lvllm {

// A workgroup per row: a wave takes one expert after the other.  Logits are fp32 sums of exact products.
template <typename T, int VEC>
__global__ __launch_bounds__(256) void moe_route_kernel(int32_t* __restrict__ ids, float* __restrict__ weights,
                                                        const typename T::store_t* __restrict__ h,
                                                        const typename T::store_t* __restrict__ w,
                                                        const float* __restrict__ bias, const MoeRouting r, const int width) {
  __shared__ float z[kMaxExperts + 1];
  const int row = blockIdx.x, lane = threadIdx.x & 63, n = r.per_row();
  const typename T::store_t* x = h + (int64_t)row * width;
  for (int e = threadIdx.x >> 6; e < r.logits(); e += 4) {
    const typename T::store_t* we = w + (int64_t)e * width;
    float acc = 0.f;
    for (int i = lane * VEC; i < width; i += 64 * VEC) {
      if constexpr (VEC == 4) {
        float a[4], b[4];
        load4<T>(x + i, a);
        load4<T>(we + i, b);
#pragma unroll
        for (int j = 0; j < 4; ++j) acc = fmaf(a[j], b[j], acc);
      } else {
        acc = fmaf(T::to_float(x[i]), T::to_float(we[i]), acc);
      }
    }
    acc = wave_sum(acc);
    if (lane == 0) z[e] = e < r.experts && bias != nullptr ? acc + bias[e] : acc;
  }
  __syncthreads();
  if (threadIdx.x < 64) choose_experts(z, r, ids + (int64_t)row * n, weights + (int64_t)row * n);
}

__global__ __launch_bounds__(1024) void moe_group_kernel(const int32_t* ids, const int total, const int per_row,
                                                         const int experts, const int shared, const MoeGroups groups) {
  group_assignments(ids, total, per_row, experts, shared, groups);
}

__global__ __launch_bounds__(256) void moe_tiles_kernel(const int experts, const int shared, const int rows, const MoeGroups groups) {
  __shared__ int count[kMaxExperts + 1], first[kMaxExperts + 2], tile0[kMaxExperts + 2];
  for (int e = threadIdx.x; e < experts; e += 256) count[e] = shared && e == experts - 1 ? rows : groups.count[e];
  __syncthreads();
  moe_running_sums(count, first, tile0, experts, groups.tile);
  __syncthreads();
  moe_write_tiles(first, tile0, experts, groups);
}

__global__ __launch_bounds__(256) void moe_slots_kernel(const int32_t* __restrict__ ids, const int total, const int per_row,
                                                        const int experts, const MoeGroups groups) {
  const int i = blockIdx.x * 256 + threadIdx.x;
  if (i >= total) return;
  const int s = min(max(groups.offsets[min(max(ids[i], 0), experts - 1)] + groups.slot[i], 0), total - 1);
  moe_place(groups, i, per_row, s);
}

int launch_moe_group(const int32_t* ids, int total, int per_row, int experts, int shared, bool counted, const MoeGroups& groups,
                     hipStream_t s) {
  if (counted) {
    hipLaunchKernelGGL(moe_tiles_kernel, dim3(1), dim3(256), 0, s, experts, shared, total / per_row, groups);
    LV_LAUNCH_CHECK();
    hipLaunchKernelGGL(moe_slots_kernel, dim3((total + 255) / 256), dim3(256), 0, s, ids, total, per_row, experts, groups);
  } else {
    hipLaunchKernelGGL(moe_group_kernel, dim3(1), dim3(1024), 0, s, ids, total, per_row, experts, shared, groups);
  }
  LV_LAUNCH_CHECK();
  return 0;
}

// 16 slots x 16 outputs a workgroup, row-major weights, 32 of K a turn through LDS.
template <typename T, int PRODUCT>
__global__ __launch_bounds__(256) void moe_simple_kernel(const MoeParams p) {
  using S = typename T::store_t;
  constexpr bool UP = PRODUCT != kMoeDown, GATED = PRODUCT == kMoeGated;
  __shared__ float sx[16][33], sg[16][33], su[GATED ? 16 : 1][33];
  const int e = p.tiles[4 * blockIdx.y];
  if (e < 0 || e >= p.experts) return;
  const int s0 = p.tiles[4 * blockIdx.y + 1], s1 = min(min(p.offsets[e + 1], s0 + 16), p.slots);
  const int ff = p.ff[e], K = UP ? p.width : ff, n0 = blockIdx.x * 16;
  if (n0 >= (UP ? ff : p.width)) return;
  const S* w = (const S*)p.w + p.w_offset[e];
  const int a = threadIdx.x >> 4, b = threadIdx.x & 15;  // slot, output
  float accg = 0.f, accu = 0.f;
  for (int k0 = 0; k0 < K; k0 += 32) {
    __syncthreads();
    for (int i = threadIdx.x; i < 16 * 32; i += 256) {
      const int r = i >> 5, k = k0 + (i & 31), s = s0 + r;
      float v = 0.f;
      if (s < s1 && k < K) {
        const int64_t row = UP ? min(max(p.token[s], 0), p.rows - 1) : s;
        v = T::to_float(((const S*)p.x)[row * (UP ? p.width : p.ff_max) + k]);
      }
      sx[r][i & 31] = v;
      const int n = GATED ? 2 * n0 + r : n0 + r;  // GATED: 16 gate rows, then 16 value rows
      sg[r][i & 31] = k < K && (UP || n < p.width) ? T::to_float(w[(int64_t)n * K + k]) : 0.f;
      if constexpr (GATED) su[r][i & 31] = k < K ? T::to_float(w[(int64_t)(n + 16) * K + k]) : 0.f;
    }
    __syncthreads();
#pragma unroll 8
    for (int k = 0; k < 32; ++k) {
      accg = fmaf(sx[a][k], sg[b][k], accg);
      if constexpr (GATED) accu = fmaf(sx[a][k], su[b][k], accu);
    }
  }
  const int s = s0 + a, n = n0 + b;
  if (s >= s1) return;
  if constexpr (GATED) {
    const float f = slot_weight_of(p, s);
    ((S*)p.out)[(int64_t)s * p.ff_max + n] = T::from_float(MoeActivation(p, e)(accg * f, accu * f));
  } else if constexpr (UP) {
    ((S*)p.out)[(int64_t)s * p.ff_max + n] = T::from_float(relu_squared_of(accg * slot_weight_of(p, s)));
  } else if (n < p.width) ((S*)p.out)[(int64_t)s * p.width + n] = T::from_float(accg);
}

}  // namespace lvllm

using namespace lvllm;

extern "C" int lvllm_moe_tile(int packed, int rows) { return moe_tile(packed != 0, rows); }

static MoeRouting routing_of(const lvllm_moe_routing& r) {
  return MoeRouting{r.experts, r.top, r.scoring, r.shared != LVLLM_MOE_NO_SHARED, r.shared == LVLLM_MOE_GATED_SHARED,
                    r.groups, r.keep, r.scale};
}

extern "C" int64_t lvllm_moe_route_workspace_bytes(const lvllm_moe_routing* routing, int rows, int width, int packed) {
  return packed ? moe_route_mfma_workspace(routing_of(*routing), rows, width) : 0;
}

extern "C" int lvllm_moe_route(int32_t* ids, float* weights, int32_t* offsets, int32_t* token, int32_t* slot,
                               float* slot_weight, int32_t* tiles, int max_tiles, const void* h, const void* w,
                               const float* bias, const lvllm_moe_routing* routing, int rows, int width, int packed,
                               void* workspace, int64_t workspace_bytes, int dtype, void* stream) {
  if (rows == 0) return 0;
  const MoeRouting r = routing_of(*routing);
  LV_CHECK(r.experts > 0 && r.experts < kMaxExperts && r.top > 0 && r.top <= r.experts, "experts: fewer than 1024, top of them");
  LV_CHECK(r.groups <= 1 || (r.groups <= kMaxGroups && r.experts % r.groups == 0 && r.keep > 0 && r.keep <= r.groups &&
                             r.keep * (r.experts / r.groups) >= r.top),
           "groups: at most 64 of equal size, as many kept as the chosen experts need");
  LV_CHECK(r.scoring == LVLLM_MOE_SOFTMAX || r.scoring == LVLLM_MOE_SIGMOID, "unknown scores");
  LV_CHECK((int64_t)rows * (r.top + 1) < ((int64_t)1 << 31) && max_tiles > 0, "too many assignments");
  LV_CHECK(workspace_bytes >= lvllm_moe_route_workspace_bytes(routing, rows, width, packed), "workspace too small");
  hipStream_t s = (hipStream_t)stream;
  const MoeGroups groups{offsets, token, slot, tiles, (int32_t*)workspace, moe_tile(packed != 0, rows), max_tiles, weights,
                         slot_weight};
  if (packed) {
    LV_CHECK(moe_takes_mfma(width, dtype), "packed router: bf16, a width that is a multiple of 32");
    return launch_moe_route_mfma(ids, weights, h, w, bias, r, rows, width, groups, (float*)workspace, s);
  }
  LV_DISPATCH_F32_BF16(dtype, {
    using S = typename scalar_t::store_t;
    if (width % 4 == 0)
      hipLaunchKernelGGL((moe_route_kernel<scalar_t, 4>), dim3(rows), dim3(256), 0, s, ids, weights, (const S*)h, (const S*)w,
                         bias, r, width);
    else
      hipLaunchKernelGGL((moe_route_kernel<scalar_t, 1>), dim3(rows), dim3(256), 0, s, ids, weights, (const S*)h, (const S*)w,
                         bias, r, width);
  });
  LV_LAUNCH_CHECK();
  return launch_moe_group(ids, rows * r.per_row(), r.per_row(), r.all(), r.shared, false, groups, s);
}

extern "C" int lvllm_moe_experts(void* out, const void* x, const void* w, const int64_t* w_offset, const int32_t* ff,
                                 const float* limit, const float* slot_weight, int act, const int32_t* offsets,
                                 const int32_t* token, const int32_t* tiles, int experts, int slots, int rows, int width,
                                 int ff_max, int ff_first, int ff_last, int max_tiles, int up, int packed, int dtype,
                                 void* stream) {
  if (slots == 0) return 0;
  LV_CHECK(experts > 0 && ff_max > 0 && ff_max % 32 == 0 && width > 0 && max_tiles > 0 && max_tiles <= 65535, "sizes of the experts");
  LV_CHECK(!up || act == LVLLM_MOE_SILU || act == LVLLM_MOE_RELU_SQUARED || (act == LVLLM_MOE_CLAMPED && limit != nullptr),
           "unknown activation");
  MoeParams p{};
  p.out = out; p.x = x; p.w = w; p.w_offset = w_offset; p.ff = ff; p.limit = limit; p.offsets = offsets; p.token = token;
  p.tiles = tiles; p.experts = experts; p.slots = slots; p.rows = rows; p.width = width; p.ff_max = ff_max;
  p.max_tiles = max_tiles; p.ff_first = ff_first; p.ff_last = ff_last; p.slot_weight = slot_weight; p.act = act;
  hipStream_t s = (hipStream_t)stream;
  const int product = !up ? kMoeDown : act == LVLLM_MOE_RELU_SQUARED ? kMoePlain : kMoeGated;
  if (packed) {
    LV_CHECK(moe_takes_mfma(width, dtype), "packed experts: bf16, a width that is a multiple of 32");
    return launch_moe_mfma(p, product, s);
  }
  const dim3 grid(((up ? ff_max : width) + 15) / 16, max_tiles);
  LV_DISPATCH_F32_BF16(dtype, {
    if (product == kMoeGated) hipLaunchKernelGGL((moe_simple_kernel<scalar_t, kMoeGated>), grid, dim3(256), 0, s, p);
    else if (product == kMoePlain) hipLaunchKernelGGL((moe_simple_kernel<scalar_t, kMoePlain>), grid, dim3(256), 0, s, p);
    else hipLaunchKernelGGL((moe_simple_kernel<scalar_t, kMoeDown>), grid, dim3(256), 0, s, p);
  });
  LV_LAUNCH_CHECK();
  return 0;
}
