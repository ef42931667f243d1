// Causal softmax attention over a paged cache whose key and value sizes differ, without positions in the scores, for
// gfx950.  Every sequence of a step is a chunk of query_len >= 1 new tokens that ends its context (their keys and
// values are in the cache already); query t of a chunk sits at position pos = seq_len - query_len + t and sees keys
// low(pos) .. pos and those before keep_first.  low(pos): pos - window + 1 (window > 0), the start of the aligned run of
// `chunk` positions it lies in (chunk > 0), the larger of both, or 0.  Sequences of fewer than min_query_len query tokens
// are left to the caller.
//
//   query       [rows, heads, kpad]                                (padding beyond the key size is zero)
//   key_cache   [num_blocks, kv_heads, kpad / x, block_size, x],   x = 16 / sizeof(T)
//   value_cache [num_blocks, kv_heads, vpad, block_size]
//   out         row r, head h at r * out_stride + h * vdim:  T(attention * sigmoid(gate[r, h]) * out_scale)
//
// Scores are scale * (q . k), with softcap > 0 then softcap * tanh(score / softcap).  sink[h], where given, is one more
// score of the softmax, without a key.
//
// maps = 2: a head's query and a kv head's key are two vectors of kpad / 2 each, back to back, and make two softmaxes a, b
// over the same values; with o = a - map_weight * b the result is o / sqrt(mean(o^2) + map_eps) (mean over vdim) instead of a.
//
// Scores, softmax, accumulation and the gate are fp32.  Three bodies: head_prefill.h (chunks, 32x32 MFMAs), head_decode.h
// (up to 16 (token, head, map) columns per kv head, keys cut into shares), head_attention.hip (32-bit elements and sizes
// outside the MFMA bodies' envelope).
#pragma once
#include "common.h"

namespace lvllm {

struct HeadAttnParams {
  void* out;
  const void *q, *k_cache, *v_cache, *gate;  // gate null: no gate
  const int32_t *block_tables, *seq_lens, *query_start_loc;
  float *part_o, *part_ml;  // decode shares: [rows, heads, maps, nsplit, vpad] and [rows, heads, maps, nsplit, 2]
  int num_seqs, rows, heads, kv_heads, kpad, vpad, vdim, max_blocks, block_size, max_block, nsplit;
  int max_query_len, max_seq_len, window, chunk, keep_first, maps, min_query_len;
  const float* sink;  // null: none
  float scale, out_scale, softcap, map_weight, map_eps;
  int64_t out_stride, gate_stride, k_block_stride, v_block_stride;
};

// Sequences with at most this many (token, head, map) columns per kv head, and every sequence of one token, take the decode
// body.  `group`: heads times maps per kv head.
constexpr int kDecodeCols = 16;
__device__ __forceinline__ bool takes_decode_body(int qlen, int group) { return qlen == 1 || qlen * group <= kDecodeCols; }

// low(pos)
__device__ __forceinline__ int first_seen(const HeadAttnParams& p, int pos) {
  int low = p.window > 0 ? max(0, pos - p.window + 1) : 0;
  if (p.chunk > 0) low = max(low, pos - pos % p.chunk);
  return low;
}
__device__ __forceinline__ bool sees(const HeadAttnParams& p, int key, int pos, int low) {
  return key <= pos && (key >= low || key < p.keep_first);
}

constexpr float kLog2e = 1.4426950408889634f;
// q . k -> the score times log2(e)
struct ScoreScale {
  float mul, cap;  // cap > 0: cap * tanh(mul * x) (mul for the exponential of the tanh)
  __device__ __forceinline__ explicit ScoreScale(const HeadAttnParams& p)
      : mul(p.softcap > 0.f ? 2.f * kLog2e * p.scale / p.softcap : p.scale * kLog2e), cap(p.softcap * kLog2e) {}
  __device__ __forceinline__ float capped(float x) const {  // 1 - 2 / (e^2y + 1): exact limits on both sides
    return cap - 2.f * cap * __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(mul * x));
  }
};
// what a sink adds to a softmax row's sum, for a row maximum m (times log2(e))
__device__ __forceinline__ float sink_term(const HeadAttnParams& p, int head, float m) {
  return p.sink != nullptr ? exp2f(p.sink[head] * kLog2e - m) : 0.f;
}

template <typename T>
__device__ __forceinline__ float gate_of(const HeadAttnParams& p, int64_t row, int head) {
  if (p.gate == nullptr) return p.out_scale;
  const float z = T::to_float(((const typename T::store_t*)p.gate)[row * p.gate_stride + head]);
  return p.out_scale / (1.f + expf(-z));
}

typedef __bf16 h_bf16x8_t __attribute__((ext_vector_type(8)));
typedef short h_s16x4_t __attribute__((ext_vector_type(4)));
typedef float h_f32x4_t __attribute__((ext_vector_type(4)));
typedef float h_f32x16_t __attribute__((ext_vector_type(16)));
typedef unsigned int h_u32x4_t __attribute__((ext_vector_type(4)));

__device__ __forceinline__ uint32_t pack_bf16(float a, float b) {
  return (uint32_t)BF16::from_float(a) | ((uint32_t)BF16::from_float(b) << 16);
}

// bf16, block size 16, sizes of takes_mfma (head_attention.hip)
int launch_head_prefill(const HeadAttnParams& p, hipStream_t s);
int launch_head_decode(const HeadAttnParams& p, hipStream_t s);
int launch_head_prefill_maps(const HeadAttnParams& p, hipStream_t s);
int launch_head_decode_maps(const HeadAttnParams& p, hipStream_t s);

}  // namespace lvllm
