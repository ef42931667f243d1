// The per-head RMS norm and gate behind a recurrence's read-out.
#pragma once
#include "row_ops.h"

namespace lvllm {

__device__ __forceinline__ float sigmoid_f(float z) { return 1.f / (1.f + expf(-z)); }

// Per head: o / rms(o) * weight * silu(gate) * scale -> T (SILU), or with sigmoid(gate).  o is the fp32 read-out of a recurrent state.
// weight_head_stride: 0 (one weight of size vdim for all heads) or vdim; weight null: none.  L lanes per (row, head).
template <typename T, int L, int VEC, bool SILU>
static __global__ __launch_bounds__(256) void head_norm_gate_kernel(
    typename T::store_t* __restrict__ out, const int64_t out_stride, const float* __restrict__ o,
    const typename T::store_t* __restrict__ gate, const int64_t gate_stride, const float* __restrict__ weight,
    const int weight_head_stride, const float eps, const float scale, const int rows, const int heads, const int vdim) {
  const int lane = threadIdx.x % L;
  const int64_t item = (int64_t)blockIdx.x * (256 / L) + threadIdx.x / L;
  if (item >= (int64_t)rows * heads) return;
  const int64_t row = item / heads;
  const int h = (int)(item - row * heads);
  const float* src = o + item * vdim;
  float f[VEC], z[VEC];
  float ss = 0.f;
  for (int d = lane * VEC; d < vdim; d += L * VEC) {
    load_vec<F32, VEC>(src + d, f);
#pragma unroll
    for (int j = 0; j < VEC; ++j) ss += f[j] * f[j];
  }
  const float r = 1.f / sqrtf(group_sum<L>(ss) / vdim + eps);
  for (int d = lane * VEC; d < vdim; d += L * VEC) {
    load_vec<F32, VEC>(src + d, f);
    load_vec<T, VEC>(gate + row * gate_stride + h * vdim + d, z);
#pragma unroll
    for (int j = 0; j < VEC; ++j)
      f[j] = f[j] * r * (weight != nullptr ? weight[h * weight_head_stride + d + j] : 1.f) * (SILU ? z[j] * sigmoid_f(z[j]) : sigmoid_f(z[j])) * scale;
    store_vec<T, VEC>(out + row * out_stride + h * vdim + d, f);
  }
}

template <bool SILU>
static int launch_head_norm_gate(void* out, int64_t out_stride, const float* o, const void* gate, int64_t gate_stride,
                                 const float* weight, int weight_head_stride, float eps, float scale, int rows,
                                 int heads, int vdim, int dtype, hipStream_t stream) {
  if (rows == 0) return 0;
  const int64_t items = (int64_t)rows * heads;
  const int esize = dtype == LVLLM_F32 ? 4 : 2;
  const bool vec = ((vdim | out_stride | gate_stride) & 3) == 0 && ((uintptr_t)o & 15) == 0 &&
                   (((uintptr_t)out | (uintptr_t)gate) & (4 * esize - 1)) == 0;
  const int lanes = lanes_for(vdim, vec ? 4 : 1);
  const dim3 grid((unsigned)((items * lanes + 255) / 256));
  LV_DISPATCH_DTYPE(dtype, {
    using S = scalar_t::store_t;
    LV_LANES(lanes, {
      if (vec)
        hipLaunchKernelGGL((head_norm_gate_kernel<scalar_t, kL, 4, SILU>), grid, dim3(256), 0, stream, (S*)out,
                           out_stride, o, (const S*)gate, gate_stride, weight, weight_head_stride, eps, scale, rows, heads, vdim);
      else
        hipLaunchKernelGGL((head_norm_gate_kernel<scalar_t, kL, 1, SILU>), grid, dim3(256), 0, stream, (S*)out,
                           out_stride, o, (const S*)gate, gate_stride, weight, weight_head_stride, eps, scale, rows, heads, vdim);
    })
  });
  LV_LAUNCH_CHECK();
  return 0;
}

}  // namespace lvllm
