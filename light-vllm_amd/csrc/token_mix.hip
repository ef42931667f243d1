// Row-wise operators of hybrid decoders for gfx950: the fp32 residual add with a Dynamic-Tanh norm, the token shift with
// its per-projection mixes, and squared ReLU.
//
// The residual stream and the norms are fp32; what a projection reads is rounded to its element type T once,
// when it is stored.  A step's rows are the new tokens of `num_seqs` sequences back to back (query_start_loc), sequence
// s ending at position seq_lens[s] - 1; rows past the last sequence are padding of a captured step.
#include "row_ops.h"

namespace lvllm {

// value i of a projection result: T values, or the fp32 split-K slabs of a decode GEMM, summed in slab order and rounded
// to T (the value the GEMM's own reduce pass would have stored)
template <typename T>
struct ProjOut {
  const typename T::store_t* y;  // null: no addend
  const float* partials;         // when set, y is unused
  int num_partials;
  int64_t partial_stride;
  __device__ __forceinline__ bool any() const { return y != nullptr || partials != nullptr; }
  __device__ __forceinline__ float at(int64_t i) const {
    if (partials != nullptr) {
      float s = 0.f;
      for (int p = 0; p < num_partials; ++p) s += partials[p * partial_stride + i];
      return T::to_float(T::from_float(s));
    }
    return y != nullptr ? T::to_float(y[i]) : 0.f;
  }
  // elements i .. i + 3 (i a multiple of 4)
  __device__ __forceinline__ void at4(int64_t i, float (&v)[4]) const {
    if (partials != nullptr) {
      v[0] = v[1] = v[2] = v[3] = 0.f;
      for (int p = 0; p < num_partials; ++p) {
        const float4 a = *reinterpret_cast<const float4*>(partials + p * partial_stride + i);
        v[0] += a.x; v[1] += a.y; v[2] += a.z; v[3] += a.w;
      }
#pragma unroll
      for (int j = 0; j < 4; ++j) v[j] = T::to_float(T::from_float(v[j]));
    } else if (y != nullptr) {
      load4<T>(y + i, v);
    } else {
      v[0] = v[1] = v[2] = v[3] = 0.f;
    }
  }
};

__device__ __forceinline__ float dyt(float x, float alpha, float w, float b) { return tanhf(alpha * x) * w + b; }

// x_out = x_in + y;  h = T(tanh(alpha * x_out) * w + b).  x_out may be x_in, or null when nothing is added.
template <typename T, int VEC>
__global__ void add_dyt_kernel(float* x_out, const float* x_in, const ProjOut<T> y,
                               typename T::store_t* __restrict__ h, const float* __restrict__ alpha,
                               const float* __restrict__ w, const float* __restrict__ b, const int64_t n, const int width) {
  const int64_t i = ((int64_t)blockIdx.x * blockDim.x + threadIdx.x) * VEC;
  if (i >= n) return;
  const int c = (int)(i % width);
  const float a = alpha[0];
  if constexpr (VEC == 4) {
    float v[4];
    y.at4(i, v);
    const float4 x = *reinterpret_cast<const float4*>(x_in + i);
    v[0] += x.x; v[1] += x.y; v[2] += x.z; v[3] += x.w;
    if (x_out != nullptr) *reinterpret_cast<float4*>(x_out + i) = float4{v[0], v[1], v[2], v[3]};
    const float4 ww = *reinterpret_cast<const float4*>(w + c), bb = *reinterpret_cast<const float4*>(b + c);
    const float o[4] = {dyt(v[0], a, ww.x, bb.x), dyt(v[1], a, ww.y, bb.y), dyt(v[2], a, ww.z, bb.z), dyt(v[3], a, ww.w, bb.w)};
    store4<T>(h + i, o);
  } else {
    const float v = x_in[i] + y.at(i);
    if (x_out != nullptr) x_out[i] = v;
    h[i] = T::from_float(dyt(v, a, w[c], b[c]));
  }
}

// Residual add + Dynamic-Tanh norm + token shift: with h the normed row and h' the normed row of the token before it
// (the sequence's carried row for the first token of a portion, zeros for the first token of a sequence),
//   mix[m] = T(h + (h' - h) * mu[m]),  m = 0 .. num_mix - 1,
// and the last row's h becomes the sequence's carried row.  A thread owns (row, VEC columns) and derives h' from x_in
// itself, so x_out must not be x_in.  The thread of a portion's FIRST row also stores the carried row: it is the one
// that has read the old one.
template <typename T, int VEC>
__global__ void add_dyt_shift_mix_kernel(float* __restrict__ x_out, const float* __restrict__ x_in, const ProjOut<T> y,
                                         typename T::store_t* __restrict__ mix, const float* __restrict__ mu,
                                         const int num_mix, const float* __restrict__ alpha, const float* __restrict__ w,
                                         const float* __restrict__ b, float* __restrict__ carried,
                                         const int64_t carried_stride, const int32_t* __restrict__ state_slots,
                                         const int num_slots, const int32_t* __restrict__ query_start_loc,
                                         const int32_t* __restrict__ seq_lens, const int num_seqs, const int rows,
                                         const int width) {
  const int per_row = (width + blockDim.x * VEC - 1) / (blockDim.x * VEC);  // workgroups of a row
  const int row = blockIdx.x / per_row;
  const int c0 = ((blockIdx.x - row * per_row) * blockDim.x + threadIdx.x) * VEC;
  if (c0 >= width) return;
  const float a = alpha[0];
  const int64_t base = (int64_t)row * width + c0;
  const int64_t n = (int64_t)rows * width;
  float ww[VEC], bb[VEC], h[VEC], hp[VEC], xv[VEC];
#pragma unroll
  for (int j = 0; j < VEC; ++j) { ww[j] = w[c0 + j]; bb[j] = b[c0 + j]; }
  auto load_row = [&](int64_t at, float (&x)[VEC], float (&out)[VEC]) {
    if constexpr (VEC == 4) {
      y.at4(at, x);
      const float4 v = *reinterpret_cast<const float4*>(x_in + at);
      x[0] += v.x; x[1] += v.y; x[2] += v.z; x[3] += v.w;
    } else {
      x[0] = x_in[at] + y.at(at);
    }
#pragma unroll
    for (int j = 0; j < VEC; ++j) out[j] = dyt(x[j], a, ww[j], bb[j]);
  };
  load_row(base, xv, h);
  if (x_out != nullptr)
#pragma unroll
    for (int j = 0; j < VEC; ++j) x_out[base + j] = xv[j];

  const int seq = find_seq(query_start_loc, num_seqs, row);
  const int qbeg = seq < num_seqs ? query_start_loc[seq] : 0;
  if (seq >= num_seqs) {  // padding row
#pragma unroll
    for (int j = 0; j < VEC; ++j) hp[j] = 0.f;
  } else if (row > qbeg) {
    float t[VEC];
    load_row(base - width, t, hp);
  } else {
    const int qlen = query_start_loc[seq + 1] - qbeg;
    const int slot = state_slots[seq];
    const bool live = slot >= 0 && slot < num_slots;
    float* st = carried + (int64_t)(live ? slot : 0) * carried_stride + c0;
    const bool fresh = seq_lens[seq] <= qlen || !live;
#pragma unroll
    for (int j = 0; j < VEC; ++j) hp[j] = fresh ? 0.f : st[j];
    if (live) {
      float last[VEC], t[VEC];
      if (qlen > 1) {
        load_row((int64_t)(qbeg + qlen - 1) * width + c0, t, last);
      } else {
#pragma unroll
        for (int j = 0; j < VEC; ++j) last[j] = h[j];
      }
#pragma unroll
      for (int j = 0; j < VEC; ++j) st[j] = last[j];
    }
  }
  for (int m = 0; m < num_mix; ++m) {
    float o[VEC];
#pragma unroll
    for (int j = 0; j < VEC; ++j) o[j] = h[j] + (hp[j] - h[j]) * mu[m * width + c0 + j];
    if constexpr (VEC == 4) store4<T>(mix + m * n + base, o);
    else mix[m * n + base] = T::from_float(o[0]);
  }
}

// y = max(x, 0)^2 elementwise (out may be x)
template <typename T, int VEC>
__global__ void relu_squared_kernel(typename T::store_t* out, const typename T::store_t* x, const int64_t n) {
  const int64_t i = ((int64_t)blockIdx.x * blockDim.x + threadIdx.x) * VEC;
  if (i >= n) return;
  if constexpr (VEC == 8) {
    const uint4 raw = *reinterpret_cast<const uint4*>(x + i);
    const uint16_t* s = reinterpret_cast<const uint16_t*>(&raw);
    uint4 o;
    uint16_t* d = reinterpret_cast<uint16_t*>(&o);
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      d[j] = T::from_float(relu_squared_of(T::to_float(s[j])));
    }
    *reinterpret_cast<uint4*>(out + i) = o;
  } else {
    out[i] = T::from_float(relu_squared_of(T::to_float(x[i])));
  }
}

template <typename T>
static ProjOut<T> proj_out(const void* y, const float* partials, int num_partials, int64_t n) {
  return ProjOut<T>{(const typename T::store_t*)y, partials, num_partials, n};
}

}  // namespace lvllm

using namespace lvllm;

extern "C" int lvllm_add_dyt(float* x_out, const float* x_in, const void* y, const float* partials, int num_partials,
                             void* h, const float* alpha, const float* weight, const float* bias, int rows, int width,
                             int dtype, void* stream) {
  if (rows == 0) return 0;
  LV_CHECK(rows > 0 && width > 0, "rows and width must be positive");
  const int64_t n = (int64_t)rows * width;
  LV_DISPATCH_DTYPE(dtype, {
    using S = scalar_t::store_t;
    const auto p = proj_out<scalar_t>(y, partials, num_partials, n);
    if (width % 4 == 0) {
      hipLaunchKernelGGL((add_dyt_kernel<scalar_t, 4>), dim3((unsigned)((n / 4 + 255) / 256)), dim3(256), 0,
                         (hipStream_t)stream, x_out, x_in, p, (S*)h, alpha, weight, bias, n, width);
    } else {
      hipLaunchKernelGGL((add_dyt_kernel<scalar_t, 1>), dim3((unsigned)((n + 255) / 256)), dim3(256), 0,
                         (hipStream_t)stream, x_out, x_in, p, (S*)h, alpha, weight, bias, n, width);
    }
  });
  LV_LAUNCH_CHECK();
  return 0;
}

extern "C" int lvllm_add_dyt_shift_mix(float* x_out, const float* x_in, const void* y, const float* partials,
                                       int num_partials, void* mix, const float* mu, int num_mix, const float* alpha,
                                       const float* weight, const float* bias, float* carried, int64_t carried_stride,
                                       const int32_t* state_slots, int num_slots, const int32_t* query_start_loc,
                                       const int32_t* seq_lens, int num_seqs, int rows, int width, int dtype, void* stream) {
  if (rows == 0) return 0;
  LV_CHECK(rows > 0 && width > 0 && num_mix > 0, "positive rows, width and mixes");
  LV_CHECK(x_out != x_in, "x_out must not be x_in: neighbouring rows read x_in");
  LV_CHECK((y == nullptr && partials == nullptr) || x_out != nullptr, "an addend needs x_out");
  LV_DISPATCH_DTYPE(dtype, {
    using S = scalar_t::store_t;
    const auto p = proj_out<scalar_t>(y, partials, num_partials, (int64_t)rows * width);
    if (width % 4 == 0) {
      hipLaunchKernelGGL((add_dyt_shift_mix_kernel<scalar_t, 4>), dim3((unsigned)rows * ((width + 1023) / 1024)), dim3(256), 0,
                         (hipStream_t)stream, x_out, x_in, p, (S*)mix, mu, num_mix, alpha, weight, bias, carried,
                         carried_stride, state_slots, num_slots, query_start_loc, seq_lens, num_seqs, rows, width);
    } else {
      hipLaunchKernelGGL((add_dyt_shift_mix_kernel<scalar_t, 1>), dim3((unsigned)rows * ((width + 255) / 256)), dim3(256), 0,
                         (hipStream_t)stream, x_out, x_in, p, (S*)mix, mu, num_mix, alpha, weight, bias, carried,
                         carried_stride, state_slots, num_slots, query_start_loc, seq_lens, num_seqs, rows, width);
    }
  });
  LV_LAUNCH_CHECK();
  return 0;
}

extern "C" int lvllm_relu_squared(void* out, const void* x, int64_t n, int dtype, void* stream) {
  if (n == 0) return 0;
  hipStream_t s = (hipStream_t)stream;
  const bool vec = dtype != LVLLM_F32 && n % 8 == 0 && ((((uintptr_t)out | (uintptr_t)x) & 15) == 0);
  if (vec && dtype == LVLLM_BF16) {
    hipLaunchKernelGGL((relu_squared_kernel<BF16, 8>), dim3((unsigned)((n / 8 + 255) / 256)), dim3(256), 0, s,
                       (uint16_t*)out, (const uint16_t*)x, n);
  } else if (vec) {
    hipLaunchKernelGGL((relu_squared_kernel<F16, 8>), dim3((unsigned)((n / 8 + 255) / 256)), dim3(256), 0, s,
                       (uint16_t*)out, (const uint16_t*)x, n);
  } else {
    LV_DISPATCH_DTYPE(dtype, {
      using S = scalar_t::store_t;
      hipLaunchKernelGGL((relu_squared_kernel<scalar_t, 1>), dim3((unsigned)((n + 255) / 256)), dim3(256), 0, s, (S*)out,
                         (const S*)x, n);
    });
  }
  LV_LAUNCH_CHECK();
  return 0;
}
