// Residual streams for gfx950: instead of one residual a decoder carries n of them, and a sublayer reads a weighted sum of the
// streams and writes to all of them.  One launch between two sublayers:
//   x_t = sum_s mix[s, t] x_s + out[t] y         (all t from the old streams; y: what the sublayer returned)
//   u   = sum_t in[t] x_t                        (the next sublayer's weights; behind the last one they are all 1)
//   h   = T(u * weight / sqrt(mean(u^2) + eps))
// and one for the embedding, whose row is every stream's start.  Everything is fp32; h, which projections read, is rounded to the
// element type T once.
//
// y comes as rows of T, as the fp32 split-K slabs of a decode GEMM, or as the slots of a mixture of experts: row r is
// sum_i slot_weight[r, i] * y[slot[r, i]].
#include "row_ops.h"

namespace lvllm {

constexpr int kMaxStreams = 16;

struct StreamMixParams {
  const float* x_in;      // streams in_stride apart (0: all of them are the same rows)
  float* x_out;           // may be x_in; null: not kept
  int64_t in_stride, out_stride;
  void* h;
  const void* y;
  const float* partials;
  const int32_t* slots;
  const float* slot_weights;
  const float *mix, *out, *in, *weight;  // [from, to], [streams], [streams], [width]
  int streams, num_partials, num_slots, total_slots, rows, width;
  float eps;
};

// A workgroup per row; a thread keeps its ITEMS groups of VEC columns of y and u in registers and takes the streams of one group
// after the other.  N: the number of streams, kMaxStreams: up to that many.
template <typename T, int VEC, int ITEMS, int N>
__global__ __launch_bounds__(1024) void stream_mix_kernel(const StreamMixParams p) {
  using S = typename T::store_t;
  constexpr int B = ITEMS <= 2 ? 8 : 4;  // rows in flight
  __shared__ float red[16], coef[kMaxStreams * (kMaxStreams + 2)];
  const int row = blockIdx.x, n = N == kMaxStreams ? p.streams : N;
  const int64_t base = (int64_t)row * p.width;
  auto column = [&](int it) { return (it * (int)blockDim.x + (int)threadIdx.x) * VEC; };
  for (int i = threadIdx.x; i < n * (n + 2); i += blockDim.x)
    coef[i] = i < n * n ? p.mix[i] : i < n * n + n ? p.out[i - n * n] : p.in[i - n * n - n];
  constexpr bool kAhead = N < kMaxStreams && ITEMS == 1;  // streams asked for before y
  float first[kAhead ? N : 1][VEC];
  if constexpr (kAhead) {
#pragma unroll
    for (int s = 0; s < N; ++s)
      if (column(0) < p.width) load_vec<F32, VEC>(p.x_in + s * p.in_stride + base + column(0), first[s]);
  }
  float y[ITEMS][VEC], ss = 0.f;
#pragma unroll
  for (int it = 0; it < ITEMS; ++it)
#pragma unroll
    for (int j = 0; j < VEC; ++j) y[it][j] = 0.f;
  auto add_rows = [&](int count, auto weight_of, auto load) __attribute__((always_inline)) {
    for (int i0 = 0; i0 < count; i0 += B) {
      float w[B];
#pragma unroll
      for (int i = 0; i < B; ++i) w[i] = i0 + i < count ? weight_of(i0 + i) : 0.f;
#pragma unroll
      for (int it = 0; it < ITEMS; ++it) {
        if (column(it) >= p.width) continue;
        float t[B][VEC];
#pragma unroll
        for (int i = 0; i < B; ++i)
          if (i0 + i < count) load(i0 + i, column(it), t[i]);
#pragma unroll
        for (int i = 0; i < B; ++i)
          if (i0 + i < count) {
#pragma unroll
            for (int j = 0; j < VEC; ++j) y[it][j] = fmaf(w[i], t[i][j], y[it][j]);
          }
      }
    }
  };
  if (p.slots != nullptr) {
    const int32_t* slots = p.slots + (int64_t)row * p.num_slots;
    const float* weights = p.slot_weights + (int64_t)row * p.num_slots;
    add_rows(p.num_slots, [&](int i) { return weights[i]; }, [&](int i, int c, float (&t)[VEC]) {
      load_vec<T, VEC>((const S*)p.y + (int64_t)min(max(slots[i], 0), p.total_slots - 1) * p.width + c, t);
    });
  } else if (p.partials != nullptr) {
    add_rows(p.num_partials, [](int) { return 1.f; }, [&](int i, int c, float (&t)[VEC]) {
      load_vec<F32, VEC>(p.partials + (int64_t)i * p.rows * p.width + base + c, t);
    });
  } else {
#pragma unroll
    for (int it = 0; it < ITEMS; ++it)
      if (column(it) < p.width) load_vec<T, VEC>((const S*)p.y + base + column(it), y[it]);
  }
  __syncthreads();
  const float *out = coef + n * n, *in = out + n;
#pragma unroll
  for (int it = 0; it < ITEMS; ++it) {
    const int c = column(it);
    if (c >= p.width) continue;
    float x[N][VEC], u[VEC];
#pragma unroll
    for (int s = 0; s < N; ++s) {
      if (N == kMaxStreams && s >= n) continue;
      if constexpr (kAhead) {
#pragma unroll
        for (int j = 0; j < VEC; ++j) x[s][j] = first[s][j];
      } else {
        load_vec<F32, VEC>(p.x_in + s * p.in_stride + base + c, x[s]);
      }
    }
#pragma unroll
    for (int j = 0; j < VEC; ++j) u[j] = 0.f;
#pragma unroll
    for (int t = 0; t < N; ++t) {
      if (N == kMaxStreams && t >= n) continue;
      float v[VEC];
#pragma unroll
      for (int j = 0; j < VEC; ++j) v[j] = out[t] * y[it][j];
#pragma unroll
      for (int s = 0; s < N; ++s) {
        if (N == kMaxStreams && s >= n) continue;
#pragma unroll
        for (int j = 0; j < VEC; ++j) v[j] = fmaf(coef[s * n + t], x[s][j], v[j]);
      }
      if (p.x_out != nullptr) store_vec<F32, VEC>(p.x_out + t * p.out_stride + base + c, v);
#pragma unroll
      for (int j = 0; j < VEC; ++j) u[j] = fmaf(in[t], v[j], u[j]);
    }
#pragma unroll
    for (int j = 0; j < VEC; ++j) {
      y[it][j] = u[j];
      ss = fmaf(u[j], u[j], ss);
    }
  }
  const float f = 1.f / sqrtf(block_sum(ss, red) / (float)p.width + p.eps);
#pragma unroll
  for (int it = 0; it < ITEMS; ++it) {
    if (column(it) >= p.width) continue;
    float w[VEC];
    load_vec<F32, VEC>(p.weight + column(it), w);
#pragma unroll
    for (int j = 0; j < VEC; ++j) w[j] *= y[it][j] * f;
    store_vec<T, VEC>((S*)p.h + base + column(it), w);
  }
}

// x = table[token] (what every stream starts as), h = T(norm of x * sum(in))
template <typename T, int VEC, int ITEMS>
__global__ __launch_bounds__(1024) void stream_embed_kernel(float* __restrict__ x, typename T::store_t* __restrict__ h,
                                                            const typename T::store_t* __restrict__ table,
                                                            const int64_t* __restrict__ ids, const float* __restrict__ in,
                                                            const int streams, const float* __restrict__ weight, const float eps,
                                                            const int vocab, const int width) {
  __shared__ float red[16];
  const int row = blockIdx.x;
  const int64_t id = min(max(ids[row], (int64_t)0), (int64_t)vocab - 1), base = (int64_t)row * width;
  float total = 0.f;
  for (int s = 0; s < streams; ++s) total += in[s];
  auto column = [&](int it) { return (it * (int)blockDim.x + (int)threadIdx.x) * VEC; };
  float v[ITEMS][VEC], ss = 0.f;
#pragma unroll
  for (int it = 0; it < ITEMS; ++it) {
    const int c = column(it);
    if (c >= width) continue;
    load_vec<T, VEC>(table + id * width + c, v[it]);
    store_vec<F32, VEC>(x + base + c, v[it]);
#pragma unroll
    for (int j = 0; j < VEC; ++j) {
      v[it][j] *= total;
      ss = fmaf(v[it][j], v[it][j], ss);
    }
  }
  const float f = 1.f / sqrtf(block_sum(ss, red) / (float)width + eps);
#pragma unroll
  for (int it = 0; it < ITEMS; ++it) {
    const int c = column(it);
    if (c >= width) continue;
    float w[VEC];
    load_vec<F32, VEC>(weight + c, w);
#pragma unroll
    for (int j = 0; j < VEC; ++j) w[j] *= v[it][j] * f;
    store_vec<T, VEC>(h + base + c, w);
  }
}

template <typename T, int VEC, int ITEMS>
static void launch_mix(const StreamMixParams& p, int threads, hipStream_t s) {
  const dim3 grid(p.rows), block(threads);
  switch (p.streams) {
    case 2: hipLaunchKernelGGL((stream_mix_kernel<T, VEC, ITEMS, 2>), grid, block, 0, s, p); break;
    case 3: hipLaunchKernelGGL((stream_mix_kernel<T, VEC, ITEMS, 3>), grid, block, 0, s, p); break;
    case 4: hipLaunchKernelGGL((stream_mix_kernel<T, VEC, ITEMS, 4>), grid, block, 0, s, p); break;
    default: hipLaunchKernelGGL((stream_mix_kernel<T, VEC, ITEMS, kMaxStreams>), grid, block, 0, s, p);
  }
}

}  // namespace lvllm

using namespace lvllm;

extern "C" int lvllm_stream_mix(float* x_out, int64_t out_stride, const float* x_in, int64_t in_stride, void* h, const void* y,
                                const float* partials, int num_partials, const int32_t* slots, const float* slot_weights,
                                int num_slots, int total_slots, const float* mix, const float* out, const float* in, int streams,
                                const float* weight, float eps, int rows, int width, int dtype, void* stream) {
  if (rows == 0) return 0;
  LV_CHECK(streams >= 1 && streams <= kMaxStreams, "1 .. 16 streams");
  LV_CHECK(y != nullptr || partials != nullptr, "no sublayer output");
  LV_CHECK(slots == nullptr || (y != nullptr && slot_weights != nullptr && total_slots > 0), "slots without their rows");
  StreamMixParams p{};
  p.x_in = x_in; p.x_out = x_out; p.in_stride = in_stride; p.out_stride = out_stride; p.h = h; p.y = y; p.partials = partials;
  p.num_partials = num_partials; p.slots = slots; p.slot_weights = slot_weights; p.num_slots = num_slots;
  p.total_slots = total_slots; p.mix = mix; p.out = out; p.in = in; p.weight = weight; p.streams = streams; p.rows = rows;
  p.width = width; p.eps = eps;
  hipStream_t s = (hipStream_t)stream;
  const int threads = threads_of(rows, width % 4 == 0 ? width / 4 : width);
#define LV_GO(VEC_, ITEMS_) LV_DISPATCH_F32_BF16(dtype, (launch_mix<scalar_t, VEC_, ITEMS_>(p, threads, s)))
  LV_ROWS(width, threads, LV_GO)
#undef LV_GO
  LV_LAUNCH_CHECK();
  return 0;
}

extern "C" int lvllm_stream_embed(float* x, void* h, const void* table, const int64_t* ids, const float* in, int streams,
                                  const float* weight, float eps, int rows, int vocab, int width, int dtype, void* stream) {
  if (rows == 0) return 0;
  LV_CHECK(vocab > 0 && width > 0 && streams >= 1, "an empty table or no stream");
  hipStream_t s = (hipStream_t)stream;
  const int threads = threads_of(rows, width % 4 == 0 ? width / 4 : width);
#define LV_GO(VEC_, ITEMS_)                                                                                              \
  LV_DISPATCH_F32_BF16(dtype, {                                                                                          \
    using S = typename scalar_t::store_t;                                                                                \
    hipLaunchKernelGGL((stream_embed_kernel<scalar_t, VEC_, ITEMS_>), dim3(rows), dim3(threads), 0, s, x, (S*)h,         \
                       (const S*)table, ids, in, streams, weight, eps, vocab, width);                                    \
  })
  LV_ROWS(width, threads, LV_GO)
#undef LV_GO
  LV_LAUNCH_CHECK();
  return 0;
}
