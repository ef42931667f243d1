// Row-wise operators of hybrid decoders for gfx950: the fp32 residual add with a Dynamic-Tanh norm, the token shift with
// its per-projection mixes, squared ReLU, per-head query/key RMS norms with the paged-cache write, and the gates in
// front of an output projection.
//
// The residual stream, the norms and every gate are fp32; what a projection reads is rounded to its element type T once,
// when it is stored.  A step's rows are the new tokens of `num_seqs` sequences back to back (query_start_loc), sequence
// s ending at position seq_lens[s] - 1; rows past the last sequence are padding of a captured step.
#include "common.h"

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

// VEC consecutive elements <-> floats
template <typename T, int VEC>
__device__ __forceinline__ void load_vec(const typename T::store_t* p, float (&v)[VEC]) {
  if constexpr (VEC == 8) {
    static_assert(sizeof(typename T::store_t) == 2, "16-byte pieces of 16-bit elements");
    const uint4 a = *reinterpret_cast<const uint4*>(p);
    const uint32_t w[4] = {a.x, a.y, a.z, a.w};
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      v[2 * j] = T::to_float((uint16_t)w[j]);
      v[2 * j + 1] = T::to_float((uint16_t)(w[j] >> 16));
    }
  } else if constexpr (VEC == 4) {
    load4<T>(p, v);
  } else {
    v[0] = T::to_float(p[0]);
  }
}
template <typename T, int VEC>
__device__ __forceinline__ void store_vec(typename T::store_t* p, const float (&v)[VEC]) {
  if constexpr (VEC == 8) {
    uint32_t w[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) w[j] = (uint32_t)T::from_float(v[2 * j]) | ((uint32_t)T::from_float(v[2 * j + 1]) << 16);
    *reinterpret_cast<uint4*>(p) = uint4{w[0], w[1], w[2], w[3]};
  } else if constexpr (VEC == 4) {
    store4<T>(p, v);
  } else {
    p[0] = T::from_float(v[0]);
  }
}
template <int L>
__device__ __forceinline__ float group_sum(float v) {  // over L neighbouring lanes
#pragma unroll
  for (int m = L / 2; m >= 1; m >>= 1) v += __shfl_xor(v, m);
  return v;
}

// Per-head RMS norm of queries and keys (weights [dim], shared by the heads) and the write of the normed keys and the
// values into a paged cache whose key and value sizes differ:
//   key_cache   [num_blocks, kv_heads, kpad / x, block_size, x],  x = 16 / sizeof(T), kpad >= dim (rest zeroed)
//   value_cache [num_blocks, kv_heads, vpad, block_size],         vpad >= vdim (rest zeroed)
// q_out [rows, heads, kpad] (padding zeroed).  L lanes per (row, head); the values of few rows ride along as further
// "heads" (with_values), those of many go through value_cache_tile_kernel.
template <typename T, int L, int VEC>
__global__ __launch_bounds__(256) void qk_norm_cache_kernel(
    typename T::store_t* __restrict__ q_out, typename T::store_t* __restrict__ key_cache,
    typename T::store_t* __restrict__ value_cache, const typename T::store_t* __restrict__ q,
    const typename T::store_t* __restrict__ k, const typename T::store_t* __restrict__ v, const int64_t row_stride,
    const float* __restrict__ q_weight, const float* __restrict__ k_weight, const float eps, const int rows, const int heads,
    const int kv_heads, const int dim, const int vdim, const int kpad, const int vpad, const bool with_values,
    const int64_t* __restrict__ slot_mapping, const int64_t num_slots, const int block_size, const int64_t k_block_stride,
    const int64_t v_block_stride) {
  using S = typename T::store_t;
  constexpr int x = 16 / sizeof(S);
  const int lane = threadIdx.x % L;
  const int per_row = heads + (with_values ? 2 : 1) * kv_heads;
  const unsigned item = blockIdx.x * (256 / L) + threadIdx.x / L;
  const int row = (int)(item / (unsigned)per_row), h = (int)(item - (unsigned)row * per_row);
  if (row >= rows) return;
  int64_t block = 0;
  int off = 0;
  if (h >= heads) {
    const int64_t slot = slot_mapping[row];
    if (slot < 0 || slot >= num_slots) return;
    block = slot / block_size;
    off = (int)(slot - block * block_size);
  }
  if (h >= heads + kv_heads) {
    const int g = h - heads - kv_heads;
    const S* src = v + row * row_stride + (int64_t)g * vdim;
    S* dst = value_cache + block * v_block_stride + (int64_t)g * vpad * block_size + off;
    for (int d = lane; d < vpad; d += L) dst[(int64_t)d * block_size] = d < vdim ? src[d] : T::from_float(0.f);
    return;
  }
  const bool is_q = h < heads;
  const S* src = (is_q ? q + (int64_t)h * dim : k + (int64_t)(h - heads) * dim) + row * row_stride;
  const float* wt = is_q ? q_weight : k_weight;
  S* dst = is_q ? q_out + ((int64_t)row * heads + h) * kpad
                : key_cache + block * k_block_stride + (int64_t)(h - heads) * kpad * block_size + (int64_t)off * x;
  float f[VEC];
  float ss = 0.f;
  for (int d = lane * VEC; d < dim; d += L * VEC) {
    load_vec<T, VEC>(src + d, f);
#pragma unroll
    for (int j = 0; j < VEC; ++j) ss += f[j] * f[j];
  }
  const bool one_pass = dim <= L * VEC;  // (the values are still in registers)
  const float r = 1.f / sqrtf(group_sum<L>(ss) / dim + eps);
  for (int d = lane * VEC; d < kpad; d += L * VEC) {
    float o[VEC];
    if (d < dim) {
      if (!one_pass) load_vec<T, VEC>(src + d, f);
#pragma unroll
      for (int j = 0; j < VEC; ++j) o[j] = f[j] * r * wt[d + j];
    } else {
#pragma unroll
      for (int j = 0; j < VEC; ++j) o[j] = 0.f;
    }
    store_vec<T, VEC>(is_q ? dst + d : dst + (int64_t)(d / x) * block_size * x + d % x, o);
  }
}

// Values of many rows: a workgroup takes 64 rows of one kv head through LDS.  Its rows are cut into groups of consecutive
// slots inside one aligned 8-slot window; a thread stores a (d, group) as one piece when the group is full.
constexpr int kValueTile = 64;
template <typename S>
__global__ __launch_bounds__(256) void value_cache_tile_kernel(S* __restrict__ value_cache, const S* __restrict__ v,
                                                               const int64_t row_stride, const int rows, const int vdim,
                                                               const int vpad, const int64_t* __restrict__ slot_mapping,
                                                               const int64_t num_slots, const int block_size,
                                                               const int64_t v_block_stride) {
  struct alignas(16) Eight { S e[8]; };
  constexpr int LD = kValueTile + 2;
  extern __shared__ __attribute__((aligned(16))) char smem[];
  S* tile = reinterpret_cast<S*>(smem);  // [vdim][LD]
  __shared__ int64_t slots[kValueTile];
  __shared__ int groups[kValueTile], num_groups;  // first row | length << 8
  const int row0 = blockIdx.x * kValueTile, head = blockIdx.y, nt = min(kValueTile, rows - row0), tid = threadIdx.x;
  if (tid < kValueTile) {
    int64_t s = tid < nt ? slot_mapping[row0 + tid] : -1;
    if (s >= num_slots) s = -1;
    slots[tid] = s;
    const int64_t prev = (int64_t)__shfl_up((long long)s, 1);
    const bool first = s >= 0 && (tid == 0 || prev < 0 || s != prev + 1 || (s & 7) == 0);
    const uint64_t starts = __ballot(first), used = __ballot(s >= 0);
    if (first) {
      const uint64_t above = tid == 63 ? 0 : (starts | ~used) >> (tid + 1);
      const int len = above ? __builtin_ctzll(above) + 1 : 64 - tid;
      groups[__builtin_popcountll(starts & ((1ull << tid) - 1))] = tid | (len << 8);
    }
    if (tid == 0) num_groups = __builtin_popcountll(starts);
  }
  const S* src = v + (int64_t)row0 * row_stride + (int64_t)head * vdim;
  for (int i = tid; i < nt * vdim; i += 256) {
    const int t = i / vdim, d = i - t * vdim;
    tile[d * LD + t] = src[t * row_stride + d];
  }
  __syncthreads();
  const int ng = num_groups;
  for (int i = tid; i < vpad * ng; i += 256) {
    const int d = i / ng, gr = groups[i - d * ng], t = gr & 0xff, len = gr >> 8;
    const int64_t s = slots[t], b = s / block_size;
    S* dst = value_cache + b * v_block_stride + ((int64_t)head * vpad + d) * block_size + (s - b * block_size);
    Eight e;
#pragma unroll
    for (int j = 0; j < 8; ++j) e.e[j] = (d < vdim && j < len) ? tile[d * LD + t + j] : (S)0;
    if (len == 8) {
      *reinterpret_cast<Eight*>(dst) = e;
    } else {
#pragma unroll
      for (int j = 0; j < 8; ++j)
        if (j < len) dst[j] = e.e[j];
    }
  }
}

__device__ __forceinline__ float sigmoid_f(float z) { return 1.f / (1.f + expf(-z)); }

// Per head: o / rms(o) * weight * silu(gate) * scale -> T.  o is the fp32 read-out of a recurrent state.
// weight_head_stride: 0 (one weight of size vdim for all heads) or vdim.  L lanes per (row, head).
template <typename T, int L, int VEC>
__global__ __launch_bounds__(256) void head_norm_gate_kernel(
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
      f[j] = f[j] * r * weight[h * weight_head_stride + d + j] * (z[j] * sigmoid_f(z[j])) * scale;
    store_vec<T, VEC>(out + row * out_stride + h * vdim + d, f);
  }
}

// lanes that cover n elements in one pass of VEC each: 8, 16, 32 or 64
static int lanes_for(int n, int vec) {
  int l = 8;
  while (l < 64 && l * vec < n) l *= 2;
  return l;
}
#define LV_LANES(LANES_, ...)                         \
  switch (LANES_) {                                   \
    case 8: { constexpr int kL = 8; __VA_ARGS__ } break;   \
    case 16: { constexpr int kL = 16; __VA_ARGS__ } break; \
    case 32: { constexpr int kL = 32; __VA_ARGS__ } break; \
    default: { constexpr int kL = 64; __VA_ARGS__ } break; \
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

extern "C" int lvllm_qk_norm_cache(void* q_out, void* key_cache, void* value_cache, const void* q, const void* k,
                                   const void* v, int64_t row_stride, const float* q_weight, const float* k_weight,
                                   float eps, int rows, int heads, int kv_heads, int dim, int vdim, int kpad, int vpad,
                                   const int64_t* slot_mapping, int64_t num_blocks, int block_size,
                                   int64_t k_block_stride, int64_t v_block_stride, int dtype, void* stream) {
  if (rows == 0) return 0;
  LV_CHECK(heads > 0 && kv_heads > 0 && heads % kv_heads == 0, "heads must be a multiple of kv_heads");
  LV_CHECK(dim <= kpad && vdim <= vpad && kpad % 8 == 0, "padded sizes must hold the real ones");
  LV_CHECK(k_block_stride >= (int64_t)kv_heads * kpad * block_size && v_block_stride >= (int64_t)kv_heads * vpad * block_size,
           "cache blocks overlap");
  const int esize = dtype == LVLLM_F32 ? 4 : 2;
  const size_t smem = (size_t)vdim * (kValueTile + 2) * esize;
  const bool tiled = rows > 64 && smem <= 64 * 1024 && block_size % 8 == 0 && ((uintptr_t)value_cache & 15) == 0 &&
                     v_block_stride * esize % 16 == 0;
  const bool vec = ((dim | row_stride) & 3) == 0 && (((uintptr_t)q | (uintptr_t)k) & (4 * esize - 1)) == 0 &&
                   (((uintptr_t)q_out | (uintptr_t)key_cache) & 15) == 0 && k_block_stride * esize % 16 == 0;
  const bool vec8 = vec && esize == 2 && ((dim | row_stride) & 7) == 0 && (((uintptr_t)q | (uintptr_t)k) & 15) == 0;
  const int64_t items = (int64_t)rows * (heads + (tiled ? 1 : 2) * kv_heads);
  LV_CHECK(items <= INT32_MAX && kv_heads <= 65535, "too many rows");
#define LV_QK(VEC_)                                                                                                          \
  hipLaunchKernelGGL((qk_norm_cache_kernel<scalar_t, kL, VEC_>), grid, dim3(256), 0, (hipStream_t)stream, (S*)q_out,          \
                     (S*)key_cache, (S*)value_cache, (const S*)q, (const S*)k, (const S*)v, row_stride, q_weight, k_weight,  \
                     eps, rows, heads, kv_heads, dim, vdim, kpad, vpad, !tiled, slot_mapping, num_blocks * block_size,       \
                     block_size, k_block_stride, v_block_stride)
  LV_DISPATCH_DTYPE(dtype, {
    using S = scalar_t::store_t;
    constexpr int kWide = sizeof(S) == 2 ? 8 : 4;  // elements of a 16-byte piece
    const int lanes = lanes_for(kpad, vec8 ? kWide : vec ? 4 : 1);
    const dim3 grid((unsigned)((items * lanes + 255) / 256));
    LV_LANES(lanes, {
      if (vec8) LV_QK(kWide);
      else if (vec) LV_QK(4);
      else LV_QK(1);
    })
    if (tiled)
      hipLaunchKernelGGL((value_cache_tile_kernel<S>), dim3((rows + kValueTile - 1) / kValueTile, kv_heads), dim3(256), smem,
                         (hipStream_t)stream, (S*)value_cache, (const S*)v, row_stride, rows, vdim, vpad, slot_mapping,
                         num_blocks * block_size, block_size, v_block_stride);
  });
#undef LV_QK
  LV_LAUNCH_CHECK();
  return 0;
}

extern "C" int lvllm_head_norm_gate(void* out, int64_t out_stride, const float* o, const void* gate, int64_t gate_stride,
                                    const float* weight, int weight_head_stride, float eps, float scale, int rows,
                                    int heads, int vdim, int dtype, void* stream) {
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
        hipLaunchKernelGGL((head_norm_gate_kernel<scalar_t, kL, 4>), grid, dim3(256), 0, (hipStream_t)stream, (S*)out,
                           out_stride, o, (const S*)gate, gate_stride, weight, weight_head_stride, eps, scale, rows, heads, vdim);
      else
        hipLaunchKernelGGL((head_norm_gate_kernel<scalar_t, kL, 1>), grid, dim3(256), 0, (hipStream_t)stream, (S*)out,
                           out_stride, o, (const S*)gate, gate_stride, weight, weight_head_stride, eps, scale, rows, heads, vdim);
    })
  });
  LV_LAUNCH_CHECK();
  return 0;
}
