// Short causal convolutions over time for gfx950, per channel, and their SiLU:
//   y[t, c] = silu(sum_j weight[taps - 1 - j, c] * x[t - j, c]),   j = 0 .. taps - 1, zeros before a sequence's start
//
// A sequence carries its last inputs in a ring of `taps` fp32 rows per slot: the input of position p is in row p mod taps.  A
// token reads the rows of the taps - 1 positions before it and writes its own, which no token of the same step reads out of the
// ring.  Nothing is ever cleared: rows of positions before 0 are not read.
#pragma once
#include "common.h"

namespace lvllm {

constexpr int kMaxTaps = 16;

__device__ __forceinline__ float silu_of(float z) { return z / (1.f + expf(-z)); }

}  // namespace lvllm
