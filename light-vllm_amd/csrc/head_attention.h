// Causal softmax attention over a paged cache whose key and value sizes differ, without positions in the scores, for
// gfx950.  Every sequence of a step is a chunk of query_len >= 1 new tokens that ends its context (their keys and
// values are in the cache already); query t of a chunk sits at position pos = seq_len - query_len + t and sees keys
// max(0, pos - window + 1) .. pos (window <= 0: keys 0 .. pos).  Sequences of fewer than min_query_len query tokens are left
// to the caller.
//
//   query       [rows, heads, kpad]                                (padding beyond the key size is zero)
//   key_cache   [num_blocks, kv_heads, kpad / x, block_size, x],   x = 16 / sizeof(T)
//   value_cache [num_blocks, kv_heads, vpad, block_size]
//   out         row r, head h at r * out_stride + h * vdim:  T(attention * sigmoid(gate[r, h]) * out_scale)
//
// Scores, softmax, accumulation and the gate are fp32.  Three bodies: head_attention_prefill.hip (chunks, 32x32 MFMAs),
// head_attention_decode.hip (up to 16 (token, head) columns per kv head, keys cut into shares), head_attention.hip
// (32-bit elements and sizes outside the MFMA bodies' envelope).
#pragma once
#include "common.h"

namespace lvllm {

struct HeadAttnParams {
  void* out;
  const void *q, *k_cache, *v_cache, *gate;  // gate null: no gate
  const int32_t *block_tables, *seq_lens, *query_start_loc;
  float *part_o, *part_ml;  // decode shares: [rows, heads, nsplit, vpad] and [rows, heads, nsplit, 2]
  int num_seqs, rows, heads, kv_heads, kpad, vpad, vdim, max_blocks, block_size, max_block, nsplit;
  int max_query_len, max_seq_len, window, min_query_len;
  float scale, out_scale;
  int64_t out_stride, gate_stride, k_block_stride, v_block_stride;
};

// Sequences with at most this many (token, head) columns per kv head, and every sequence of one token, take the decode body.
constexpr int kDecodeCols = 16;
__device__ __forceinline__ bool takes_decode_body(int qlen, int group) { return qlen == 1 || qlen * group <= kDecodeCols; }

__device__ __forceinline__ int first_seen(int pos, int window) { return window > 0 ? max(0, pos - window + 1) : 0; }

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

int launch_head_prefill(const HeadAttnParams& p, hipStream_t s);  // 16-bit (bf16), block size 16, sizes of head_sizes_ok
int launch_head_decode(const HeadAttnParams& p, hipStream_t s);

}  // namespace lvllm
