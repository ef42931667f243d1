// Rotary positions: the sine and cosine of a pair's angle.
#pragma once
#include "common.h"

namespace lvllm {

// position * turns full turns: the product is taken in double, so that far positions keep the fp32 sine's own accuracy.
__device__ __forceinline__ void rotation_of(int64_t position, double turns, float& c, float& s) {
  const double t = (double)position * turns;
  sincospif((float)(2.0 * (t - rint(t))), &s, &c);
}
// ... of a rotation that also makes vectors `grow` times as long
__device__ __forceinline__ void rotation_of(int64_t position, double turns, float grow, float& c, float& s) {
  rotation_of(position, turns, c, s);
  c *= grow;
  s *= grow;
}

}  // namespace lvllm
