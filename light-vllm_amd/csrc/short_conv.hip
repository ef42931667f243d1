// Short convolutions of portions (short_conv.h).  A thread walks 16 rows of VEC channels; the thread of a portion's first rows is
// the only one that reads the ring, and it also writes the portion's last inputs there.
#include "row_ops.h"
#include "short_conv.h"

namespace lvllm {

constexpr int kConvRows = 16;

struct ShortConvParams {
  void* out;
  const void* x;
  const float* weight;  // [taps, channels]
  float* state;         // slot s, row r, channel c at s * state_stride + r * channels + c
  const int32_t *state_slots, *query_start_loc, *seq_lens;
  int64_t out_stride, x_stride, state_stride;
  int taps, channels, num_slots;
};

// TAPS: at least the number of taps; the rows before the current one stay in registers
template <typename T, int VEC, int TAPS>
__global__ __launch_bounds__(256) void short_conv_kernel(const ShortConvParams p) {
  using S = typename T::store_t;
  const int c = (blockIdx.x * 256 + threadIdx.x) * VEC, seq = blockIdx.z, t0 = blockIdx.y * kConvRows;
  const int qbeg = p.query_start_loc[seq], qlen = p.query_start_loc[seq + 1] - qbeg;
  if (t0 >= qlen || c >= p.channels) return;
  const int ctx = p.seq_lens[seq] - qlen, slot = p.state_slots[seq];
  const bool live = slot >= 0 && slot < p.num_slots;
  float* ring = p.state + (int64_t)(live ? slot : 0) * p.state_stride + c;
  const S* x = (const S*)p.x + qbeg * p.x_stride + c;
  float w[TAPS][VEC], v[TAPS][VEC];  // v[j]: the input j rows back
#pragma unroll
  for (int j = 0; j < TAPS; ++j)
#pragma unroll
    for (int i = 0; i < VEC; ++i) w[j][i] = v[j][i] = 0.f;
#pragma unroll
  for (int j = 0; j < TAPS; ++j) {
    if (j >= p.taps) continue;
    load_vec<F32, VEC>(p.weight + (int64_t)(p.taps - 1 - j) * p.channels + c, w[j]);
    const int t = t0 - 1 - j;  // becomes v[j + 1] in the first turn
    if (j + 1 >= p.taps) continue;
    if (t >= 0) load_vec<T, VEC>(x + t * p.x_stride, v[j]);
    else if (live && ctx + t >= 0) load_vec<F32, VEC>(ring + (int64_t)((ctx + t) % p.taps) * p.channels, v[j]);
  }
  const int n = min(kConvRows, qlen - t0);
  S* out = (S*)p.out + (int64_t)(qbeg + t0) * p.out_stride + c;
  constexpr int B = 4;  // rows in flight
  for (int r0 = 0; r0 < n; r0 += B) {
    float next[B][VEC];
#pragma unroll
    for (int r = 0; r < B; ++r) load_vec<T, VEC>(x + min(t0 + r0 + r, qlen - 1) * p.x_stride, next[r]);
#pragma unroll
    for (int r = 0; r < B; ++r) {
      if (r0 + r >= n) break;
      float y[VEC];
#pragma unroll
      for (int i = 0; i < VEC; ++i) {
#pragma unroll
        for (int j = TAPS - 1; j > 0; --j) v[j][i] = v[j - 1][i];
        v[0][i] = next[r][i];
        y[i] = 0.f;
#pragma unroll
        for (int j = TAPS - 1; j >= 0; --j) y[i] = fmaf(w[j][i], v[j][i], y[i]);
        y[i] = silu_of(y[i]);
      }
      store_vec<T, VEC>(out + (r0 + r) * p.out_stride, y);
    }
  }
  if (t0 > 0 || !live) return;
  for (int t = max(0, qlen - p.taps); t < qlen; ++t) {
    float y[VEC];
    load_vec<T, VEC>(x + t * p.x_stride, y);
    store_vec<F32, VEC>(ring + (int64_t)((ctx + t) % p.taps) * p.channels, y);
  }
}

}  // namespace lvllm

using namespace lvllm;

extern "C" int lvllm_short_conv(void* out, int64_t out_stride, const void* x, int64_t x_stride, const float* weight, int taps,
                                int channels, float* state, int64_t state_stride, const int32_t* state_slots, int num_slots,
                                const int32_t* query_start_loc, const int32_t* seq_lens, int num_seqs, int max_query_len,
                                int dtype, void* stream) {
  if (num_seqs == 0 || max_query_len == 0) return 0;
  LV_CHECK(taps >= 1 && taps <= kMaxTaps && channels > 0, "1 .. 16 taps");
  LV_CHECK(state_stride >= (int64_t)taps * channels, "state slots overlap");
  const int tiles = (max_query_len + kConvRows - 1) / kConvRows;
  LV_CHECK(num_seqs <= 65535 && tiles <= 65535, "too many sequences or too long portions");
  const ShortConvParams p{out, x, weight, state, state_slots, query_start_loc, seq_lens, out_stride, x_stride, state_stride,
                          taps, channels, num_slots};
  hipStream_t s = (hipStream_t)stream;
  const int esize = dtype == LVLLM_F32 ? 4 : 2;
  const bool vec = ((channels | out_stride | x_stride | state_stride) & 3) == 0 &&
                   (((uintptr_t)out | (uintptr_t)x) & (4 * esize - 1)) == 0 &&
                   (((uintptr_t)weight | (uintptr_t)state) & 15) == 0;
  const dim3 grid((channels / (vec ? 4 : 1) + 255) / 256, tiles, num_seqs);
#define LV_GO(VEC_, TAPS_) \
  LV_DISPATCH_F32_BF16(dtype, { hipLaunchKernelGGL((short_conv_kernel<scalar_t, VEC_, TAPS_>), grid, dim3(256), 0, s, p); })
  if (vec && taps <= 4) { LV_GO(4, 4); }
  else if (vec) { LV_GO(4, kMaxTaps); }
  else if (taps <= 4) { LV_GO(1, 4); }
  else { LV_GO(1, kMaxTaps); }
#undef LV_GO
  LV_LAUNCH_CHECK();
  return 0;
}
