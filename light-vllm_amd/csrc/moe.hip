// Mixture of experts: the router, the grouping of a step's assignments, and the plain products (moe.h; the matrix-core
// bodies are in moe_mfma.hip).
#include "moe.h"

namespace lvllm {

// A workgroup per row: a wave takes one expert after the other.  Logits are fp32 sums of exact products.
template <typename T, int VEC>
__global__ __launch_bounds__(256) void moe_route_kernel(int32_t* __restrict__ ids, float* __restrict__ weights,
                                                        const typename T::store_t* __restrict__ h,
                                                        const typename T::store_t* __restrict__ w,
                                                        const float* __restrict__ bias, const int experts, const int shared,
                                                        const int top, const int width) {
  __shared__ float z[kMaxExperts + 1];
  const int row = blockIdx.x, lane = threadIdx.x & 63, n = top + shared;
  const typename T::store_t* x = h + (int64_t)row * width;
  for (int e = threadIdx.x >> 6; e < experts + shared; e += 4) {
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
    if (lane == 0) z[e] = e < experts ? acc + bias[e] : acc;
  }
  __syncthreads();
  if (threadIdx.x < 64) choose_experts(z, experts, top, shared != 0, ids + (int64_t)row * n, weights + (int64_t)row * n);
}

// Counts, offsets, slots and tiles of `total` assignments; one workgroup.  `shared`: the last assignment of every row is the
// last expert's, in row order.
__global__ __launch_bounds__(1024) void moe_group_kernel(int32_t* __restrict__ offsets, int32_t* __restrict__ token,
                                                         int32_t* __restrict__ slot, int32_t* __restrict__ tiles,
                                                         const int32_t* __restrict__ ids, const int total, const int per_row,
                                                         const int experts, const int shared, const int tile, const int max_tiles) {
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

// 16 slots x 16 outputs a workgroup, row-major weights, 32 of K a turn through LDS.
template <typename T, bool UP>
__global__ __launch_bounds__(256) void moe_simple_kernel(const MoeParams p) {
  using S = typename T::store_t;
  __shared__ float sx[16][33], sg[16][33], su[UP ? 16 : 1][33];
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
      const int n = UP ? 2 * n0 + r : n0 + r;  // UP: 16 gate rows, then 16 value rows
      sg[r][i & 31] = k < K && (UP || n < p.width) ? T::to_float(w[(int64_t)n * K + k]) : 0.f;
      if constexpr (UP) su[r][i & 31] = k < K ? T::to_float(w[(int64_t)(n + 16) * K + k]) : 0.f;
    }
    __syncthreads();
#pragma unroll 8
    for (int k = 0; k < 32; ++k) {
      accg = fmaf(sx[a][k], sg[b][k], accg);
      if constexpr (UP) accu = fmaf(sx[a][k], su[b][k], accu);
    }
  }
  const int s = s0 + a, n = n0 + b;
  if (s >= s1) return;
  if constexpr (UP) ((S*)p.out)[(int64_t)s * p.ff_max + n] = T::from_float(clamped_gate(accg, accu, p.limit[e]));
  else if (n < p.width) ((S*)p.out)[(int64_t)s * p.width + n] = T::from_float(accg);
}

}  // namespace lvllm

using namespace lvllm;

extern "C" int lvllm_moe_route(int32_t* ids, float* weights, const void* h, const void* w, const float* bias, int experts,
                               int shared, int top, int rows, int width, int packed, int dtype, void* stream) {
  if (rows == 0) return 0;
  LV_CHECK(experts > 0 && experts < kMaxExperts && top > 0 && top <= experts && top <= 64, "experts (fewer than 1024) or top (at most 64)");
  hipStream_t s = (hipStream_t)stream;
  if (packed) {
    LV_CHECK(moe_takes_mfma(width, dtype), "packed router: bf16, a width that is a multiple of 32");
    return launch_moe_route_mfma(ids, weights, h, w, bias, experts, shared != 0, top, rows, width, s);
  }
  LV_DISPATCH_F32_BF16(dtype, {
    using S = typename scalar_t::store_t;
    if (width % 4 == 0)
      hipLaunchKernelGGL((moe_route_kernel<scalar_t, 4>), dim3(rows), dim3(256), 0, s, ids, weights, (const S*)h, (const S*)w,
                         bias, experts, shared != 0, top, width);
    else
      hipLaunchKernelGGL((moe_route_kernel<scalar_t, 1>), dim3(rows), dim3(256), 0, s, ids, weights, (const S*)h, (const S*)w,
                         bias, experts, shared != 0, top, width);
  });
  LV_LAUNCH_CHECK();
  return 0;
}

extern "C" int lvllm_moe_tile(int packed) { return packed ? kMoeTile : kMoeSimpleTile; }

extern "C" int lvllm_moe_group(int32_t* offsets, int32_t* token, int32_t* slot, int32_t* tiles, const int32_t* ids, int total,
                               int per_row, int experts, int shared, int packed, int max_tiles, void* stream) {
  if (total == 0) return 0;
  LV_CHECK(experts > 0 && experts <= kMaxExperts && per_row > 0, "experts (shared one included): at most 1024");
  hipLaunchKernelGGL(moe_group_kernel, dim3(1), dim3(1024), 0, (hipStream_t)stream, offsets, token, slot, tiles, ids, total,
                     per_row, experts, shared != 0, lvllm_moe_tile(packed), max_tiles);
  LV_LAUNCH_CHECK();
  return 0;
}

extern "C" int lvllm_moe_experts(void* out, const void* x, const void* w, const int64_t* w_offset, const int32_t* ff,
                                 const float* limit, const int32_t* offsets, const int32_t* token, const int32_t* tiles,
                                 int experts, int slots, int rows, int width, int ff_max, int ff_first, int ff_last, int max_tiles, int up,
                                 int packed, int dtype, void* stream) {
  if (slots == 0) return 0;
  LV_CHECK(experts > 0 && ff_max > 0 && ff_max % 32 == 0 && width > 0 && max_tiles > 0 && max_tiles <= 65535, "sizes of the experts");
  MoeParams p{};
  p.out = out; p.x = x; p.w = w; p.w_offset = w_offset; p.ff = ff; p.limit = limit; p.offsets = offsets; p.token = token;
  p.tiles = tiles; p.experts = experts; p.slots = slots; p.rows = rows; p.width = width; p.ff_max = ff_max;
  p.max_tiles = max_tiles; p.ff_first = ff_first; p.ff_last = ff_last;
  hipStream_t s = (hipStream_t)stream;
  if (packed) {
    LV_CHECK(moe_takes_mfma(width, dtype), "packed experts: bf16, a width that is a multiple of 32");
    return launch_moe_mfma(p, up != 0, s);
  }
  const dim3 grid(((up ? ff_max : width) + 15) / 16, max_tiles);
  LV_DISPATCH_F32_BF16(dtype, {
    if (up) hipLaunchKernelGGL((moe_simple_kernel<scalar_t, true>), grid, dim3(256), 0, s, p);
    else hipLaunchKernelGGL((moe_simple_kernel<scalar_t, false>), grid, dim3(256), 0, s, p);
  });
  LV_LAUNCH_CHECK();
  return 0;
}
