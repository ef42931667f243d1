// Row-wise operators of decoders that norm what a sublayer returns (not what it reads), for gfx950: the scaled embedding,
// and one launch for
//   v     = x + y * gain / sqrt(mean(y^2) + eps)          y: the sublayer's output
//   x_out = sum_j weight[j] * stream[j] + weight[n] * v     (optional: the weighted average over the depth)
//   h     = T(x_out), or T(x_out * out_gain / sqrt(mean(x_out^2) + eps))
// Everything is fp32; h, which projections read, is rounded to the element type T once.
//
// y comes as rows of T, as the fp32 split-K slabs of a decode GEMM, or as the slots of a mixture of experts: row r is
// sum_i slot_weight[r, i] * y[slot[r, i]].
#include "row_ops.h"

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

// A workgroup per row; a thread keeps its ITEMS groups of VEC columns in registers.  Everything that does not depend on the
// norm -- the sublayer's output, the stream, the earlier streams -- is read before the reduction, several rows at a time.
template <typename T, int VEC, int ITEMS>
__global__ __launch_bounds__(1024) void norm_add_mix_kernel(const DepthMixParams p) {
  using S = typename T::store_t;
  constexpr int B = ITEMS <= 2 ? 8 : 4;  // rows in flight
  __shared__ float red[16];
  const int row = blockIdx.x;
  const int64_t base = (int64_t)row * p.width;
  auto column = [&](int it) { return (it * (int)blockDim.x + (int)threadIdx.x) * VEC; };
  float v[ITEMS][VEC], x[ITEMS][VEC], mix[ITEMS][VEC];
#pragma unroll
  for (int it = 0; it < ITEMS; ++it) {
#pragma unroll
    for (int j = 0; j < VEC; ++j) v[it][j] = x[it][j] = mix[it][j] = 0.f;
    if (column(it) < p.width) load_vec<F32, VEC>(p.x_in + base + column(it), x[it]);
  }
  auto add_rows = [&](float (&acc)[ITEMS][VEC], int n, auto weight_of, auto load) __attribute__((always_inline)) {
    for (int i0 = 0; i0 < n; i0 += B) {
      float w[B];
#pragma unroll
      for (int i = 0; i < B; ++i) w[i] = i0 + i < n ? weight_of(i0 + i) : 0.f;
#pragma unroll
      for (int it = 0; it < ITEMS; ++it) {
        if (column(it) >= p.width) continue;
        float t[B][VEC];
#pragma unroll
        for (int i = 0; i < B; ++i)
          if (i0 + i < n) load(i0 + i, column(it), t[i]);
#pragma unroll
        for (int i = 0; i < B; ++i)
          if (i0 + i < n) {
#pragma unroll
            for (int j = 0; j < VEC; ++j) acc[it][j] = fmaf(w[i], t[i][j], acc[it][j]);
          }
      }
    }
  };
  if (p.slots != nullptr) {
    const int32_t* slots = p.slots + (int64_t)row * p.num_slots;
    const float* weights = p.slot_weights + (int64_t)row * p.num_slots;
    add_rows(v, p.num_slots, [&](int i) { return weights[i]; }, [&](int i, int c, float (&t)[VEC]) {
      load_vec<T, VEC>((const S*)p.y + (int64_t)min(max(slots[i], 0), p.total_slots - 1) * p.width + c, t);
    });
  } else if (p.partials != nullptr) {
    add_rows(v, p.num_partials, [](int) { return 1.f; }, [&](int i, int c, float (&t)[VEC]) {
      load_vec<F32, VEC>(p.partials + (int64_t)i * p.rows * p.width + base + c, t);
    });
  } else {
#pragma unroll
    for (int it = 0; it < ITEMS; ++it)
      if (column(it) < p.width) load_vec<T, VEC>((const S*)p.y + base + column(it), v[it]);
  }
  if (p.weights != nullptr)
    add_rows(mix, p.num_streams, [&](int i) { return p.weights[i]; }, [&](int i, int c, float (&t)[VEC]) {
      load_vec<F32, VEC>(p.streams + i * p.stream_stride + base + c, t);
    });
  float ss = 0.f;
#pragma unroll
  for (int it = 0; it < ITEMS; ++it)
#pragma unroll
    for (int j = 0; j < VEC; ++j) ss = fmaf(v[it][j], v[it][j], ss);
  ss = block_sum(ss, red);
  const float f = p.gain[0] / sqrtf(ss / (float)p.width + p.eps);
  const float wv = p.weights != nullptr ? p.weights[p.num_streams] : 1.f;
  float so = 0.f;
#pragma unroll
  for (int it = 0; it < ITEMS; ++it) {
    if (column(it) >= p.width) continue;
#pragma unroll
    for (int j = 0; j < VEC; ++j) x[it][j] = fmaf(v[it][j], f, x[it][j]);
    if (p.v_out != nullptr) store_vec<F32, VEC>(p.v_out + base + column(it), x[it]);
#pragma unroll
    for (int j = 0; j < VEC; ++j) {
      v[it][j] = fmaf(wv, x[it][j], mix[it][j]);
      so = fmaf(v[it][j], v[it][j], so);
    }
    if (p.x_out != nullptr) store_vec<F32, VEC>(p.x_out + base + column(it), v[it]);
  }
  float fo = 1.f;
  if (p.out_gain != nullptr) {
    so = block_sum(so, red);
    fo = p.out_gain[0] / sqrtf(so / (float)p.width + p.out_eps);
  }
#pragma unroll
  for (int it = 0; it < ITEMS; ++it) {
    if (column(it) >= p.width) continue;
#pragma unroll
    for (int j = 0; j < VEC; ++j) v[it][j] *= fo;
    store_vec<T, VEC>((S*)p.h + base + column(it), v[it]);
  }
}

// x = table[id] * scale, h = T(x)
template <typename T, int VEC>
__global__ __launch_bounds__(256) void embed_scale_kernel(float* __restrict__ x, typename T::store_t* __restrict__ h,
                                                          const typename T::store_t* __restrict__ table,
                                                          const int64_t* __restrict__ ids, const float scale, const int vocab,
                                                          const int width) {
  const int row = blockIdx.x;
  const int64_t id = ids[row] < 0 ? 0 : ids[row] >= vocab ? vocab - 1 : ids[row];
  const int64_t base = (int64_t)row * width;
  for (int c = threadIdx.x * VEC; c < width; c += 256 * VEC) {
    float v[VEC];
    load_vec<T, VEC>(table + id * width + c, v);
#pragma unroll
    for (int j = 0; j < VEC; ++j) v[j] *= scale;
    store_vec<F32, VEC>(x + base + c, v);
    store_vec<T, VEC>(h + base + c, v);
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
    if (width % 4 == 0)
      hipLaunchKernelGGL((embed_scale_kernel<scalar_t, 4>), dim3(rows), dim3(256), 0, (hipStream_t)stream, x, (S*)h,
                         (const S*)table, ids, scale, vocab, width);
    else
      hipLaunchKernelGGL((embed_scale_kernel<scalar_t, 1>), dim3(rows), dim3(256), 0, (hipStream_t)stream, x, (S*)h,
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
  // few rows: as many threads as a row has groups of columns; many: 256, several groups each
  const int vec = width % 4 == 0 ? 4 : 1, groups = width / vec;
  int threads = 256;
  while (threads < 1024 && (rows <= 256 ? threads < groups : threads * 4 < groups)) threads *= 2;
  const int items = (groups + threads - 1) / threads;
#define LV_GO(VEC_, ITEMS_)                                                                                        \
  LV_DISPATCH_F32_BF16(dtype, {                                                                                    \
    hipLaunchKernelGGL((norm_add_mix_kernel<scalar_t, VEC_, ITEMS_>), dim3(rows), dim3(threads), 0, s, p);         \
  })
  if (vec == 4) {
    if (items <= 1) { LV_GO(4, 1); }
    else if (items <= 2) { LV_GO(4, 2); }
    else {
      LV_CHECK(items <= 4, "rows of at most 16384");
      LV_GO(4, 4);
    }
  } else {
    LV_CHECK(width <= 4096, "rows that are no multiple of 4: at most 4096");
    LV_GO(1, 4);
  }
#undef LV_GO
  LV_LAUNCH_CHECK();
  return 0;
}
