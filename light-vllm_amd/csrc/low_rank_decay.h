// ln w [rows, channels] from a low-rank projection (log_decay.h), on fp32 MFMAs.
#pragma once
#include "log_decay.h"

namespace lvllm {

// A workgroup per 64 rows x 128 channels; f(u) through LDS, a wave's two tiles of 16 channels against all four row tiles.
constexpr int kDecayRows = 64, kDecayCols = 128;
template <typename T>
static __global__ __launch_bounds__(256) void log_decay_kernel(float* __restrict__ out, const typename T::store_t* __restrict__ u,
                                                        const int64_t u_stride, const float* __restrict__ a_t,  // [rank, channels]
                                                        const float* __restrict__ bias, const int kind,
                                                        const float inv_tau, const float* __restrict__ scale,
                                                        const int rows, const int rank, const int channels) {
  extern __shared__ float su[];  // [kDecayRows][ld]
  const int rank4 = (rank + 3) & ~3, ld = rank4 + 1;
  const int row0 = blockIdx.y * kDecayRows, nr = min(kDecayRows, rows - row0);
  for (int k = threadIdx.x & 63; k < rank4; k += 64) {
    constexpr int N = kDecayRows / 4;
    const int r0 = threadIdx.x >> 6;
    typename T::store_t raw[N];  // (all of a thread's loads in flight at once)
#pragma unroll
    for (int i = 0; i < N; ++i) raw[i] = u[(int64_t)(row0 + min(r0 + 4 * i, nr - 1)) * u_stride + min(k, rank - 1)];
#pragma unroll
    for (int i = 0; i < N; ++i) {
      const float f = k < rank ? T::to_float(raw[i]) : 0.f;
      su[(r0 + 4 * i) * ld + k] = kind == kDecayNegExp ? tanhf(f) : f;
    }
  }
  __syncthreads();
  const int lane = threadIdx.x & 63, g = lane >> 4, c = lane & 15;
  const int ch0 = blockIdx.x * kDecayCols + __builtin_amdgcn_readfirstlane(threadIdx.x >> 6) * 32 + c;
  const float* b0 = a_t + min(ch0, channels - 1);
  const float* b1 = a_t + min(ch0 + 16, channels - 1);
  r_f32x4_t z[2][4];
#pragma unroll
  for (int j = 0; j < 2; ++j)
#pragma unroll
    for (int i = 0; i < 4; ++i) z[j][i] = r_f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll 8
  for (int k0 = 0; k0 < rank4; k0 += 4) {
    const int64_t at = (int64_t)min(k0 + g, rank - 1) * channels;  // (beyond the rank: f(u) is zero)
    const float x0 = b0[at], x1 = b1[at];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const float a = su[(16 * i + c) * ld + k0 + g];
      z[0][i] = mfma_f32(a, x0, z[0][i]);
      z[1][i] = mfma_f32(a, x1, z[1][i]);
    }
  }
#pragma unroll
  for (int j = 0; j < 2; ++j) {
    const int ch = ch0 + 16 * j;
    if (ch >= channels) continue;
    const float bb = bias[ch], f = scale != nullptr ? scale[ch] : inv_tau;
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int row = 16 * i + 4 * g + r;
        if (row < nr) out[(int64_t)(row0 + row) * channels + ch] = log_decay_of(z[j][i][r] + bb, kind, f);
      }
  }
}

// `scale` [channels] of softplus decays, or null: inv_tau
static int launch_log_decay(float* out, const void* u, int64_t u_stride, const float* a_t, const float* bias, int kind,
                            float inv_tau, const float* scale, int rows, int rank, int channels, int dtype, hipStream_t s) {
  if (rows == 0) return 0;
  LV_CHECK(rank > 0 && rank <= 512 && channels > 0, "rank must be in 1 .. 512");
  const size_t smem = (size_t)kDecayRows * (((rank + 3) & ~3) + 1) * 4;
  const int ny = (rows + kDecayRows - 1) / kDecayRows;
  LV_CHECK(ny <= 65535, "too many rows");
  LV_DISPATCH_DTYPE(dtype, {
    using S = scalar_t::store_t;
    if (smem > 64 * 1024)
      (void)hipFuncSetAttribute((const void*)log_decay_kernel<scalar_t>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)smem);
    hipLaunchKernelGGL((log_decay_kernel<scalar_t>), dim3((channels + kDecayCols - 1) / kDecayCols, ny), dim3(256), smem, s, out,
                       (const S*)u, u_stride, a_t, bias, kind, inv_tau, scale, rows, rank, channels);
  });
  LV_LAUNCH_CHECK();
  return 0;
}

}  // namespace lvllm
