// Row-wise operators of decoders that norm what a sublayer returns (not what it reads), for gfx950: the scaled embedding,
// and one launch for
//   v     = x + y * gain / sqrt(mean(y^2) + eps)          y: the sublayer's output
//   x_out = sum_j weight[j] * stream[j] + weight[n] * v     (optional: the weighted average over the depth)
//   h     = T(x_out), or T(x_out * out_gain / sqrt(mean(x_out^2) + eps))
// Everything is fp32; h, which projections read, is rounded to the element type T once.
//
// y comes as rows of T, as the fp32 split-K slabs of a decode GEMM, or as the slots of a mixture of experts: row r is
// sum_i slot_weight[r, i] * y[slot[r, i]].
#include "common.h"

namespace lvllm {

struct DepthMixParams {
  const float* x_in;
  float *x_out, *v_out;           // v_out: where v is kept as a stream of its own (null: not kept)
  void* h;
  const void* y;
  const float* partials;
  const int32_t* slots;
  const float* slot_weights;
  const float *gain, *out_gain;   // device scalars; out_gain null: h is x_out
  const float *streams, *weights; // weights null: x_out = v
  int64_t stream_stride;
  int num_partials, num_slots, total_slots, num_streams, rows, width;
  float eps, out_eps;
};

template <typename T, int VEC>
__device__ __forceinline__ void load_items(const typename T::store_t* p, float (&v)[VEC]) {
  if constexpr (VEC == 4) load4<T>(p, v);
  else v[0] = T::to_float(p[0]);
}
template <int VEC>
__device__ __forceinline__ void load_f32(const float* p, float (&v)[VEC]) {
  load_items<F32, VEC>(p, v);
}
template <typename T, int VEC>
__device__ __forceinline__ void store_items(typename T::store_t* p, const float (&v)[VEC]) {
  if constexpr (VEC == 4) store4<T>(p, v);
  else p[0] = T::from_float(v[0]);
}

// A workgroup per row; a thread keeps its ITEMS groups of VEC columns in registers.
template <typename T, int VEC, int ITEMS>
__global__ __launch_bounds__(256) void norm_add_mix_kernel(const DepthMixParams p) {
  using S = typename T::store_t;
  __shared__ float red[16];
  const int row = blockIdx.x;
  const int64_t base = (int64_t)row * p.width;
  float v[ITEMS][VEC];
  float ss = 0.f;
#pragma unroll
  for (int it = 0; it < ITEMS; ++it) {
    const int c = (it * 256 + threadIdx.x) * VEC;
#pragma unroll
    for (int j = 0; j < VEC; ++j) v[it][j] = 0.f;
    if (c >= p.width) continue;
    if (p.slots != nullptr) {
      for (int i = 0; i < p.num_slots; ++i) {
        const int s = min(max(p.slots[(int64_t)row * p.num_slots + i], 0), p.total_slots - 1);
        const float w = p.slot_weights[(int64_t)row * p.num_slots + i];
        float t[VEC];
        load_items<T, VEC>((const S*)p.y + (int64_t)s * p.width + c, t);
#pragma unroll
        for (int j = 0; j < VEC; ++j) v[it][j] = fmaf(w, t[j], v[it][j]);
      }
    } else if (p.partials != nullptr) {
      for (int s = 0; s < p.num_partials; ++s) {
        float t[VEC];
        load_f32<VEC>(p.partials + (int64_t)s * p.rows * p.width + base + c, t);
#pragma unroll
        for (int j = 0; j < VEC; ++j) v[it][j] += t[j];
      }
    } else {
      load_items<T, VEC>((const S*)p.y + base + c, v[it]);
    }
#pragma unroll
    for (int j = 0; j < VEC; ++j) ss = fmaf(v[it][j], v[it][j], ss);
  }
  ss = block_sum(ss, red);
  const float f = p.gain[0] / sqrtf(ss / (float)p.width + p.eps);
  const float wv = p.weights != nullptr ? p.weights[p.num_streams] : 1.f;
  float so = 0.f;
#pragma unroll
  for (int it = 0; it < ITEMS; ++it) {
    const int c = (it * 256 + threadIdx.x) * VEC;
    if (c >= p.width) continue;
    float x[VEC];
    load_f32<VEC>(p.x_in + base + c, x);
#pragma unroll
    for (int j = 0; j < VEC; ++j) x[j] = fmaf(v[it][j], f, x[j]);
    if (p.v_out != nullptr) store_items<F32, VEC>(p.v_out + base + c, x);
#pragma unroll
    for (int j = 0; j < VEC; ++j) v[it][j] = x[j] * wv;
    if (p.weights != nullptr) {
      for (int s = 0; s < p.num_streams; ++s) {
        float t[VEC];
        load_f32<VEC>(p.streams + s * p.stream_stride + base + c, t);
        const float w = p.weights[s];
#pragma unroll
        for (int j = 0; j < VEC; ++j) v[it][j] = fmaf(w, t[j], v[it][j]);
      }
    }
#pragma unroll
    for (int j = 0; j < VEC; ++j) so = fmaf(v[it][j], v[it][j], so);
    if (p.x_out != nullptr) store_items<F32, VEC>(p.x_out + base + c, v[it]);
  }
  float fo = 1.f;
  if (p.out_gain != nullptr) {
    so = block_sum(so, red);
    fo = p.out_gain[0] / sqrtf(so / (float)p.width + p.out_eps);
  }
#pragma unroll
  for (int it = 0; it < ITEMS; ++it) {
    const int c = (it * 256 + threadIdx.x) * VEC;
    if (c >= p.width) continue;
#pragma unroll
    for (int j = 0; j < VEC; ++j) v[it][j] *= fo;
    store_items<T, VEC>((S*)p.h + base + c, v[it]);
  }
}

// x = table[id] * scale, h = T(x)
template <typename T>
__global__ __launch_bounds__(256) void embed_scale_kernel(float* __restrict__ x, typename T::store_t* __restrict__ h,
                                                          const typename T::store_t* __restrict__ table,
                                                          const int64_t* __restrict__ ids, const float scale, const int vocab,
                                                          const int width) {
  const int row = blockIdx.x;
  const int64_t id = ids[row] < 0 ? 0 : ids[row] >= vocab ? vocab - 1 : ids[row];
  for (int c = threadIdx.x; c < width; c += 256) {
    const float v = T::to_float(table[id * width + c]) * scale;
    x[(int64_t)row * width + c] = v;
    h[(int64_t)row * width + c] = T::from_float(v);
  }
}

}  // namespace lvllm

using namespace lvllm;

extern "C" int lvllm_embed_scale(float* x, void* h, const void* table, const int64_t* ids, float scale, int rows, int vocab,
                                 int width, int dtype, void* stream) {
  if (rows == 0) return 0;
  LV_CHECK(vocab > 0 && width > 0, "an empty table");
  LV_DISPATCH_F32_BF16(dtype, {
    using S = typename scalar_t::store_t;
    hipLaunchKernelGGL((embed_scale_kernel<scalar_t>), dim3(rows), dim3(256), 0, (hipStream_t)stream, x, (S*)h,
                       (const S*)table, ids, scale, vocab, width);
  });
  LV_LAUNCH_CHECK();
  return 0;
}

extern "C" int lvllm_norm_add_mix(float* x_out, float* v_out, void* h, const float* x_in, const void* y,
                                  const float* partials, int num_partials, const int32_t* slots, const float* slot_weights,
                                  int num_slots, int total_slots, const float* gain, float eps, const float* streams,
                                  int64_t stream_stride, int num_streams, const float* weights, const float* out_gain,
                                  float out_eps, int rows, int width, int dtype, void* stream) {
  if (rows == 0) return 0;
  LV_CHECK(y != nullptr || partials != nullptr, "no sublayer output");
  LV_CHECK(slots == nullptr || (y != nullptr && slot_weights != nullptr && total_slots > 0), "slots without their rows");
  DepthMixParams p{};
  p.x_in = x_in; p.x_out = x_out; p.v_out = v_out; p.h = h; p.y = y; p.partials = partials; p.num_partials = num_partials;
  p.slots = slots; p.slot_weights = slot_weights; p.num_slots = num_slots; p.total_slots = total_slots; p.gain = gain;
  p.eps = eps; p.streams = streams; p.stream_stride = stream_stride; p.num_streams = num_streams; p.weights = weights;
  p.out_gain = out_gain; p.out_eps = out_eps; p.rows = rows; p.width = width;
  hipStream_t s = (hipStream_t)stream;
#define LV_GO(VEC_, ITEMS_)                                                                                        \
  LV_DISPATCH_F32_BF16(dtype, {                                                                                       \
    hipLaunchKernelGGL((norm_add_mix_kernel<scalar_t, VEC_, ITEMS_>), dim3(rows), dim3(256), 0, s, p);             \
  })
  if (width % 4 == 0) {
    const int items = (width + 1023) / 1024;
    if (items <= 1) { LV_GO(4, 1); }
    else if (items <= 2) { LV_GO(4, 2); }
    else if (items <= 4) { LV_GO(4, 4); }
    else if (items <= 8) { LV_GO(4, 8); }
    else {
      LV_CHECK(items <= 16, "rows of at most 16384");
      LV_GO(4, 16);
    }
  } else {
    LV_CHECK(width <= 4096, "rows that are no multiple of 4: at most 4096");
    if (width <= 1024) { LV_GO(1, 4); }
    else { LV_GO(1, 16); }
  }
#undef LV_GO
  LV_LAUNCH_CHECK();
  return 0;
}
