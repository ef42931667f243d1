// Helpers of row-wise operators: pieces of VEC elements, sums over groups of lanes, lanes per row.
#pragma once
#include "common.h"

namespace lvllm {

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

// lanes that cover n elements in one pass of VEC each: 8, 16, 32 or 64
inline int lanes_for(int n, int vec) {
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

// Launches of a workgroup per row whose threads keep groups of columns in registers.
// few or short rows: as many threads as a row has groups of columns; many long ones: 256, several groups each
inline int threads_of(int rows, int groups) {
  int threads = 256;
  while (threads < 1024 && (rows <= 256 || groups <= 512 ? threads < groups : threads * 4 < groups)) threads *= 2;
  return threads;
}

// vectors of 4 up to rows of 16384, single columns up to 4096
#define LV_ROWS(WIDTH_, THREADS_, GO_)                                       \
  if ((WIDTH_) % 4 == 0) {                                                   \
    const int items = ((WIDTH_) / 4 + (THREADS_) - 1) / (THREADS_);          \
    LV_CHECK(items <= 4, "rows of at most 16384");                           \
    if (items <= 1) { GO_(4, 1); }                                           \
    else if (items <= 2) { GO_(4, 2); }                                      \
    else { GO_(4, 4); }                                                      \
  } else {                                                                   \
    LV_CHECK((WIDTH_) <= 4 * (THREADS_), "rows that are no multiple of 4: at most 4096"); \
    GO_(1, 4);                                                               \
  }

}  // namespace lvllm
