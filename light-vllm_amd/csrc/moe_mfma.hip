// The products of moe.h on 16x16x32 bf16 MFMAs over packed weights: W rows are the A operand, slots the columns, so that a
// lane ends up with consecutive outputs of one slot, and gate and value of an activation in the same register of two tiles.
//
//   * few slots per expert (decode steps): bound by the weights' bytes.  A workgroup takes 16 slots of one expert and a share
//     of its outputs; the slots' rows sit in LDS in fragment order, every wave streams W tiles of its own (1 KiB a load, eight
//     k-steps in flight behind the eight in use) and needs no other wave;
//   * prompts: 128 slots x 256 W rows a workgroup, a wave 128 x 64.  The slots' rows go through LDS (two stages of 64 k,
//     XOR-swizzled), W comes from global memory straight into the operand registers of the one wave that uses it.
#include "moe.h"

namespace lvllm {

typedef __bf16 e_bf16x8_t __attribute__((ext_vector_type(8)));
typedef float e_f32x4_t __attribute__((ext_vector_type(4)));
typedef unsigned int e_u32x4_t __attribute__((ext_vector_type(4)));

__device__ __forceinline__ e_f32x4_t moe_mfma(e_u32x4_t a, e_u32x4_t b, e_f32x4_t c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(e_bf16x8_t, a), __builtin_bit_cast(e_bf16x8_t, b), c, 0, 0,
                                                 0);
}

constexpr int kStreamMaxRows = 64, kStreamMaxK = 4096, kStreamBatch = 8;

// grid (shares of the outputs, experts, groups of 16 slots)
template <bool UP>
__global__ __launch_bounds__(256, 2) void moe_stream_kernel(const MoeParams p) {
  extern __shared__ __attribute__((aligned(16))) char sx[];  // [K / 32][4][16][8]
  constexpr int NW = UP ? 2 : 1;  // W tiles of a unit: gate and value
  const int e = blockIdx.y;
  const int s0 = p.offsets[e] + 16 * blockIdx.z, s1 = min(p.offsets[e + 1], p.slots);
  if (s0 >= s1) return;
  const int lane = threadIdx.x & 63;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int g = lane >> 4, c = lane & 15;
  const int ff = p.ff[e], K = UP ? p.width : ff, steps = K >> 5;
  const int units = UP ? ff >> 4 : p.width >> 4;
  const uint16_t* w = (const uint16_t*)p.w + p.w_offset[e] + lane * 8;
  e_u32x4_t a[2][NW][kStreamBatch];
  auto fetch = [&](int u, int b, e_u32x4_t (&t)[NW][kStreamBatch]) __attribute__((always_inline)) {
#pragma unroll
    for (int j = 0; j < kStreamBatch; ++j)
#pragma unroll
      for (int i = 0; i < NW; ++i)
        if (b + j < steps) t[i][j] = *reinterpret_cast<const e_u32x4_t*>(w + ((int64_t)(NW * u + i) * steps + b + j) * 512);
  };
  int u = blockIdx.x * 4 + wave;
  if (u < units) fetch(u, 0, a[0]);
  {
    const int64_t ld = UP ? p.width : p.ff_max;
    const int slot = s0 + (threadIdx.x & 15);
    const int64_t row = slot >= s1 ? -1 : UP ? min(max(p.token[slot], 0), p.rows - 1) : slot;
    const uint16_t* x = (const uint16_t*)p.x + (row < 0 ? 0 : row) * ld;
    for (int i = threadIdx.x; i < K * 2; i += 256) {  // 16-byte chunk i: slot i % 16, entries 8 (i / 16) ..
      e_u32x4_t v{0, 0, 0, 0};
      if (row >= 0) v = *reinterpret_cast<const e_u32x4_t*>(x + (i >> 4) * 8);
      *reinterpret_cast<e_u32x4_t*>(sx + i * 16) = v;
    }
  }
  __syncthreads();
  const char* xf = sx + lane * 16;
  for (; u < units; u += gridDim.x * 4) {
    const int un = u + gridDim.x * 4;
    e_f32x4_t acc[NW];
#pragma unroll
    for (int i = 0; i < NW; ++i) acc[i] = e_f32x4_t{0.f, 0.f, 0.f, 0.f};
    auto use = [&](int b, const e_u32x4_t (&t)[NW][kStreamBatch]) __attribute__((always_inline)) {
#pragma unroll
      for (int j = 0; j < kStreamBatch; ++j)
        if (b + j < steps) {
          const e_u32x4_t x = *reinterpret_cast<const e_u32x4_t*>(xf + (b + j) * 1024);
#pragma unroll
          for (int i = 0; i < NW; ++i) acc[i] = moe_mfma(t[i][j], x, acc[i]);
        }
    };
    for (int b = 0; b < steps; b += 2 * kStreamBatch) {
      const bool two = b + kStreamBatch < steps;
      if (two) fetch(u, b + kStreamBatch, a[1]);
      use(b, a[0]);
      if (b + 2 * kStreamBatch < steps) fetch(u, b + 2 * kStreamBatch, a[0]);
      else if (un < units) fetch(un, 0, a[0]);
      if (two) use(b + kStreamBatch, a[1]);
    }
    const int slot = s0 + c;
    if (slot >= s1) continue;
    float v[4];
    if constexpr (UP) {
      const float limit = p.limit[e];
#pragma unroll
      for (int r = 0; r < 4; ++r) v[r] = clamped_gate(acc[0][r], acc[1][r], limit);
      store4<BF16>((uint16_t*)p.out + (int64_t)slot * p.ff_max + 16 * u + 4 * g, v);
    } else {
#pragma unroll
      for (int r = 0; r < 4; ++r) v[r] = acc[0][r];
      store4<BF16>((uint16_t*)p.out + (int64_t)slot * p.width + 16 * u + 4 * g, v);
    }
  }
}

// grid (blocks of 256 W rows, tiles of 128 slots)
template <bool UP>
__global__ __launch_bounds__(256, 2) void moe_tile_kernel(const MoeParams p) {
  constexpr int MT = kMoeTile / 16;
  __shared__ __attribute__((aligned(16))) char sx[2][kMoeTile * 128];
  const int e = p.tiles[2 * blockIdx.y];
  if (e < 0 || e >= p.experts) return;
  const int s0 = p.tiles[2 * blockIdx.y + 1], s1 = min(min(p.offsets[e + 1], s0 + kMoeTile), p.slots);
  const int ff = p.ff[e], K = UP ? p.width : ff, steps = K >> 5;
  const int ntiles = UP ? ff >> 3 : p.width >> 4;  // of 16 W rows
  if ((int)blockIdx.x * 16 >= ntiles || s0 >= s1) return;
  const int lane = threadIdx.x & 63;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int g = lane >> 4, c = lane & 15;
  const int nt0 = blockIdx.x * 16 + wave * 4;
  const int64_t ld = UP ? p.width : p.ff_max;
  // chunks this thread moves: row 32 i + tid / 8 of the tile, 16 bytes tid % 8 of its 128
  const int q = threadIdx.x & 7, r0 = threadIdx.x >> 3;
  const uint16_t* xrow[4];
  char* xdst[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int r = 32 * i + r0, slot = min(s0 + r, s1 - 1);
    const int64_t row = UP ? min(max(p.token[slot], 0), p.rows - 1) : slot;
    xrow[i] = (const uint16_t*)p.x + row * ld + q * 8;
    xdst[i] = sx[0] + r * 128 + ((q ^ (r & 7)) * 16);
  }
  const uint16_t* w = (const uint16_t*)p.w + p.w_offset[e] + lane * 8;
  e_u32x4_t xs[4], a[2][4][2];
  const e_u32x4_t zero{0, 0, 0, 0};
  auto fetch_x = [&](int s) __attribute__((always_inline)) {
#pragma unroll
    for (int i = 0; i < 4; ++i)
      xs[i] = s * 32 + q * 8 < K ? *reinterpret_cast<const e_u32x4_t*>(xrow[i] + s * 32) : zero;
  };
  auto put_x = [&](int stage) __attribute__((always_inline)) {
#pragma unroll
    for (int i = 0; i < 4; ++i) *reinterpret_cast<e_u32x4_t*>(xdst[i] + stage * kMoeTile * 128) = xs[i];
  };
  auto fetch_w = [&](int s, e_u32x4_t (&t)[4][2]) __attribute__((always_inline)) {
#pragma unroll
    for (int n = 0; n < 4; ++n)
#pragma unroll
      for (int k = 0; k < 2; ++k)
        t[n][k] = s + k < steps && nt0 + n < ntiles
                      ? *reinterpret_cast<const e_u32x4_t*>(w + ((int64_t)(nt0 + n) * steps + s + k) * 512) : zero;
  };
  e_f32x4_t acc[4][MT];
#pragma unroll
  for (int n = 0; n < 4; ++n)
#pragma unroll
    for (int m = 0; m < MT; ++m) acc[n][m] = e_f32x4_t{0.f, 0.f, 0.f, 0.f};
  auto use = [&](int stage, const e_u32x4_t (&t)[4][2]) __attribute__((always_inline)) {
    const char* base = sx[stage] + c * 128;
#pragma unroll
    for (int k = 0; k < 2; ++k)
#pragma unroll
      for (int m = 0; m < MT; ++m) {
        const e_u32x4_t x = *reinterpret_cast<const e_u32x4_t*>(base + m * 2048 + (((4 * k + g) ^ (c & 7)) * 16));
#pragma unroll
        for (int n = 0; n < 4; ++n) acc[n][m] = moe_mfma(t[n][k], x, acc[n][m]);
      }
  };
  fetch_x(0);
  fetch_w(0, a[0]);
  put_x(0);
  __syncthreads();
  for (int s = 0; s < steps; s += 4) {  // two stages a turn
    const bool second = s + 2 < steps;
    if (second) { fetch_x(s + 2); fetch_w(s + 2, a[1]); }
    use(0, a[0]);
    if (second) put_x(1);
    __syncthreads();
    if (!second) break;
    const bool third = s + 4 < steps;
    if (third) { fetch_x(s + 4); fetch_w(s + 4, a[0]); }
    use(1, a[1]);
    if (third) put_x(0);
    __syncthreads();
  }
  const float limit = UP ? p.limit[e] : 0.f;
#pragma unroll
  for (int m = 0; m < MT; ++m) {
    const int slot = s0 + 16 * m + c;
    if (slot >= s1) continue;
#pragma unroll
    for (int n = 0; n < 4; n += UP ? 2 : 1) {
      if (nt0 + n >= ntiles) continue;
      float v[4];
      if constexpr (UP) {
#pragma unroll
        for (int r = 0; r < 4; ++r) v[r] = clamped_gate(acc[n][m][r], acc[n + 1][m][r], limit);
        store4<BF16>((uint16_t*)p.out + (int64_t)slot * p.ff_max + (nt0 + n) * 8 + 4 * g, v);
      } else {
#pragma unroll
        for (int r = 0; r < 4; ++r) v[r] = acc[n][m][r];
        store4<BF16>((uint16_t*)p.out + (int64_t)slot * p.width + (nt0 + n) * 16 + 4 * g, v);
      }
    }
  }
}

bool moe_takes_mfma(int width, int dtype) { return dtype == LVLLM_BF16 && width % 32 == 0; }

template <bool UP>
static void go(const MoeParams& p, hipStream_t s) {
  const int K = UP ? p.width : p.ff_max, n = UP ? p.ff_max : p.width;  // of the largest expert
  if (p.rows <= kStreamMaxRows && K <= kStreamMaxK) {
    const int smem = K * 32;
    if (smem > 64 * 1024)
      (void)hipFuncSetAttribute((const void*)moe_stream_kernel<UP>, hipFuncAttributeMaxDynamicSharedMemorySize, smem);
    const int units = n / 16;
    int shares = (units + 3) / 4;
    hipLaunchKernelGGL((moe_stream_kernel<UP>), dim3(shares, p.experts, (p.rows + 15) / 16), dim3(256), smem, s, p);
  } else {
    hipLaunchKernelGGL((moe_tile_kernel<UP>), dim3((n * (UP ? 2 : 1) + 255) / 256, p.max_tiles), dim3(256), 0, s, p);
  }
}

int launch_moe_mfma(const MoeParams& p, bool up, hipStream_t s) {
  LV_CHECK(p.experts <= 65535 && p.max_tiles <= 65535, "too many experts or tiles");
  if (up) go<true>(p, s);
  else go<false>(p, s);
  LV_LAUNCH_CHECK();
  return 0;
}

}  // namespace lvllm
