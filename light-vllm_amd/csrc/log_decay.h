// Decays of linear recurrences for gfx950: their logarithms, and sums of these over a chunk of 16 tokens.
//
//   z = A f(u) + bias,   ln w = logsigmoid(z) / tau   (f = identity),
//                        ln w = -exp(z)               (f = tanh), or
//                        ln w = -scale * softplus(z)  (f = identity)
#pragma once
#include "common.h"

namespace lvllm {

enum { kDecayLogSigmoid = 0, kDecayNegExp = 1, kDecaySoftplus = 2 };

// e^x, |x| up to a few hundred: 2^(x log2 e) with the product's rounding error put back
__device__ __forceinline__ float exp_of(float x) {
  const float t = x * 1.44269502e+0f;
  const float lo = fmaf(x, 1.44269502e+0f, -t) + x * 1.92596299e-8f;
  const float r = __builtin_amdgcn_exp2f(t);
  return fmaf(r, lo * 0.693147182f, r);
}

// `scale`: 1 / tau, or a softplus decay's factor
__device__ __forceinline__ float log_decay_of(float z, int kind, float scale) {
  if (kind == kDecayNegExp) return -exp_of(fminf(z, 9.f));  // (exp(-exp(9)) is 0: a finite logarithm keeps sums finite)
  const float small = log1pf(exp_of(-fabsf(z)));
  return kind == kDecaySoftplus ? -scale * (fmaxf(z, 0.f) + small) : (fminf(z, 0.f) - small) * scale;
}

typedef float r_f32x4_t __attribute__((ext_vector_type(4)));
__device__ __forceinline__ r_f32x4_t mfma_f32(float a, float b, r_f32x4_t c) {
  return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0);
}

constexpr int kChunk = 16;
constexpr float kMaxHalfDecay = 60.f;  // ln of the largest factor measured from the middle of a chunk

// Sums of ln w over ranges of a chunk's tokens, for the lane of channel c and tokens 4g .. 4g + 3 (l).  Every range is summed
// by itself: a difference of two running sums would lose the small decays behind a large one.
struct ChunkSums {
  float h1, h2;              // the chunk's two halves
  float read[4], left[4];    // chunk's start -> what token t reads; token t -> end
  float half_q[4], half_k[4];  // the middle of the chunk -> what token t reads; token t -> the middle
  __device__ __forceinline__ ChunkSums(const float (&l)[4], int g, int c, bool has_bonus) {
    const float upto[4] = {l[0], l[0] + l[1], (l[0] + l[1]) + l[2], (l[0] + l[1]) + (l[2] + l[3])};
    const float after[4] = {l[1] + (l[2] + l[3]), l[2] + l[3], l[3], 0.f};
    const float g0 = __shfl(upto[3], c), g1 = __shfl(upto[3], 16 + c), g2 = __shfl(upto[3], 32 + c), g3 = __shfl(upto[3], 48 + c);
    const float before_g = g == 0 ? 0.f : g == 1 ? g0 : g == 2 ? g0 + g1 : g0 + g1 + g2;
    const float after_g = g == 3 ? 0.f : g == 2 ? g3 : g == 1 ? g2 + g3 : g1 + (g2 + g3);
    const float in_half = g == 0 ? g1 : g == 3 ? g2 : 0.f;  // the group of this half between this one and the middle
    h1 = g0 + g1;
    h2 = g2 + g3;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const float upto_read = has_bonus ? (r == 0 ? 0.f : upto[r == 0 ? 0 : r - 1]) : upto[r];
      const float from_read = has_bonus ? after[r] + l[r] : after[r];
      read[r] = before_g + upto_read;
      left[r] = after[r] + after_g;
      half_q[r] = g < 2 ? -(from_read + in_half) : in_half + upto_read;
      half_k[r] = g < 2 ? after[r] + in_half : -(in_half + upto[r]);
    }
  }
};

}  // namespace lvllm
