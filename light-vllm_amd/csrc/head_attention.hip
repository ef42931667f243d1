// Causal softmax attention over a paged cache whose key and value sizes differ, without positions in the scores, for
// gfx950.  Every sequence of a step is a chunk of query_len >= 1 new tokens that ends its context (their keys and
// values are in the cache already); query t of a chunk sits at position seq_len - query_len + t and sees keys 0 .. there.
//
//   query       [rows, heads, kpad]                                (padding beyond dim is zero)
//   key_cache   [num_blocks, kv_heads, kpad / x, block_size, x],   x = 16 / sizeof(T)
//   value_cache [num_blocks, kv_heads, vpad, block_size]
//   out         [rows, heads, vpad]
//
// Scores, softmax and accumulation are fp32.
#include <float.h>

#include "common.h"

namespace lvllm {

struct HeadAttnParams {
  void* out;
  const void *q, *k_cache, *v_cache;
  const int32_t *block_tables, *seq_lens, *query_start_loc;
  int num_seqs, rows, heads, kv_heads, kpad, vpad, max_blocks, block_size, max_block;
  float scale;
  int64_t k_block_stride, v_block_stride;
};

// One workgroup per (row, head): 256 keys per round, one per thread for the scores, then one value column per thread.
template <typename T>
__global__ __launch_bounds__(256) void head_attention_simple_kernel(const HeadAttnParams p) {
  using S = typename T::store_t;
  constexpr int x = 16 / sizeof(S);
  extern __shared__ float sm[];
  float* sq = sm;               // [kpad]
  float* sp = sq + p.kpad;      // [256]
  float* sacc = sp + 256;       // [vpad]
  __shared__ float red[16];
  const int row = blockIdx.x, head = blockIdx.y;
  const int seq = find_seq(p.query_start_loc, p.num_seqs, row);
  if (seq >= p.num_seqs) return;
  const int qbeg = p.query_start_loc[seq], qlen = p.query_start_loc[seq + 1] - qbeg;
  const int n_keys = p.seq_lens[seq] - qlen + (row - qbeg) + 1;
  const int kvh = head / (p.heads / p.kv_heads);
  const int32_t* table = p.block_tables + (int64_t)seq * p.max_blocks;
  const S* q = (const S*)p.q + ((int64_t)row * p.heads + head) * p.kpad;
  for (int d = threadIdx.x; d < p.kpad; d += 256) sq[d] = T::to_float(q[d]);
  for (int d = threadIdx.x; d < p.vpad; d += 256) sacc[d] = 0.f;
  float m = -FLT_MAX, l = 0.f;
  const int bs = p.block_size;
  for (int k0 = 0; k0 < n_keys; k0 += 256) {
    __syncthreads();
    const int key = k0 + threadIdx.x;
    float score = -FLT_MAX;
    if (key < n_keys) {
      const int b = min(max(table[min(key / bs, p.max_blocks - 1)], 0), p.max_block);
      const S* kc = (const S*)p.k_cache + b * p.k_block_stride + (int64_t)kvh * p.kpad * bs + (key % bs) * x;
      float acc = 0.f;
      for (int d = 0; d < p.kpad; d += x) {
        const Vec16<T> kv = *reinterpret_cast<const Vec16<T>*>(kc + (int64_t)(d / x) * bs * x);
#pragma unroll
        for (int j = 0; j < x; ++j) acc = fmaf(sq[d + j], T::to_float(kv.v[j]), acc);
      }
      score = acc * p.scale;
    }
    float mx = wave_max(score);
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = mx;
    __syncthreads();
    const float m_new = fmaxf(m, fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3])));
    const float corr = expf(m - m_new);
    const float e = key < n_keys ? expf(score - m_new) : 0.f;
    sp[threadIdx.x] = e;
    __syncthreads();
    l = l * corr + block_sum(e, red);
    m = m_new;
    const int nk = min(256, n_keys - k0);
    for (int d = threadIdx.x; d < p.vpad; d += 256) {
      float acc = sacc[d] * corr;
      for (int j = 0; j < nk; ++j) {
        const int kk = k0 + j;
        const int b = min(max(table[min(kk / bs, p.max_blocks - 1)], 0), p.max_block);
        acc = fmaf(sp[j], T::to_float(((const S*)p.v_cache)[b * p.v_block_stride + ((int64_t)kvh * p.vpad + d) * bs + kk % bs]), acc);
      }
      sacc[d] = acc;
    }
  }
  __syncthreads();
  S* out = (S*)p.out + ((int64_t)row * p.heads + head) * p.vpad;
  for (int d = threadIdx.x; d < p.vpad; d += 256) out[d] = T::from_float(sacc[d] / l);
}

}  // namespace lvllm

using namespace lvllm;

extern "C" int lvllm_head_attention(void* out, const void* q, const void* key_cache, const void* value_cache,
                                    const int32_t* block_tables, const int32_t* seq_lens, const int32_t* query_start_loc,
                                    int num_seqs, int rows, int heads, int kv_heads, int kpad, int vpad, int max_blocks,
                                    int block_size, int64_t num_blocks, float scale, int64_t k_block_stride,
                                    int64_t v_block_stride, int dtype, void* stream) {
  if (rows == 0 || num_seqs == 0) return 0;
  LV_CHECK(heads > 0 && kv_heads > 0 && heads % kv_heads == 0, "heads must be a multiple of kv_heads");
  LV_CHECK(kpad % 8 == 0 && vpad > 0 && kpad <= 8192 && vpad <= 8192, "key rows are multiples of 8 elements");
  LV_CHECK(max_blocks > 0 && num_blocks > 0 && block_size > 0, "an empty cache");
  const HeadAttnParams p{out, q, key_cache, value_cache, block_tables, seq_lens, query_start_loc, num_seqs, rows, heads,
                         kv_heads, kpad, vpad, max_blocks, block_size, (int)(num_blocks - 1), scale, k_block_stride,
                         v_block_stride};
  LV_DISPATCH_DTYPE(dtype, {
    hipLaunchKernelGGL((head_attention_simple_kernel<scalar_t>), dim3(rows, heads), dim3(256),
                       (size_t)(kpad + 256 + vpad) * 4, (hipStream_t)stream, p);
  });
  LV_LAUNCH_CHECK();
  return 0;
}
