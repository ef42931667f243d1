// Paged attention with unequal key and value sizes: the dispatcher and the body for 32-bit elements and for sizes outside
// the MFMA bodies (see head_attention.h for the layouts).
#include <float.h>

#include "head_attention.h"

namespace lvllm {

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
  if (qlen < p.min_query_len) return;
  const int n_keys = p.seq_lens[seq] - qlen + (row - qbeg) + 1;
  S* out = (S*)p.out + row * p.out_stride + (int64_t)head * p.vdim;
  if (n_keys <= 0) {  // a padding row of a captured step
    for (int d = threadIdx.x; d < p.vdim; d += 256) out[d] = T::from_float(0.f);
    return;
  }
  const int kvh = head / (p.heads / p.kv_heads);
  const int32_t* table = p.block_tables + (int64_t)seq * p.max_blocks;
  const S* q = (const S*)p.q + ((int64_t)row * p.heads + head) * p.kpad;
  for (int d = threadIdx.x; d < p.kpad; d += 256) sq[d] = T::to_float(q[d]);
  for (int d = threadIdx.x; d < p.vpad; d += 256) sacc[d] = 0.f;
  float m = -FLT_MAX, l = 0.f;
  const int bs = p.block_size;
  for (int k0 = first_seen(n_keys - 1, p.window); k0 < n_keys; k0 += 256) {
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
  const float f = gate_of<T>(p, row, head) / l;
  for (int d = threadIdx.x; d < p.vdim; d += 256) out[d] = T::from_float(sacc[d] * f);
}

}  // namespace lvllm

using namespace lvllm;

static bool mfma_size(int n, int least) {
  return n == least || n == 64 || n == 96 || n == 128 || n == 192 || n == 256;
}

static bool takes_mfma(int kpad, int vpad, int block_size, int dtype) {
  return dtype == LVLLM_BF16 && block_size == 16 && mfma_size(kpad, 64) && mfma_size(vpad, 32);
}

// Shares the keys of a sequence are cut into: enough workgroups to fill the chip, none of under 256 keys, and none at all
// beside large prompt portions
static int decode_shares(int rows, int num_seqs, int heads, int kv_heads, int max_seq_len) {
  if (rows > 512) return 1;
  const int wgs = num_seqs * kv_heads * ((heads / kv_heads + kDecodeCols - 1) / kDecodeCols);
  int n = (1024 + wgs - 1) / wgs;
  const int most = (max_seq_len + 255) / 256;
  n = n < most ? n : most;
  return n < 1 ? 1 : n > 64 ? 64 : n;
}

extern "C" int64_t lvllm_head_attention_workspace_bytes(int rows, int num_seqs, int heads, int kv_heads, int kpad, int vpad,
                                                        int block_size, int max_seq_len, int dtype) {
  if (heads <= 0 || kv_heads <= 0 || rows <= 0 || num_seqs <= 0 || !takes_mfma(kpad, vpad, block_size, dtype)) return 0;
  const int n = decode_shares(rows, num_seqs, heads, kv_heads, max_seq_len);
  return n > 1 ? (int64_t)rows * heads * n * (vpad + 2) * 4 : 0;
}

extern "C" int lvllm_head_attention(void* out, int64_t out_stride, const void* q, const void* key_cache,
                                    const void* value_cache, const void* gate, int64_t gate_stride,
                                    const int32_t* block_tables, const int32_t* seq_lens, const int32_t* query_start_loc,
                                    int num_seqs, int rows, int heads, int kv_heads, int kpad, int vpad, int vdim,
                                    int max_blocks, int block_size, int64_t num_blocks, float scale, float out_scale,
                                    int64_t k_block_stride, int64_t v_block_stride, int max_query_len, int max_seq_len,
                                    int window, int min_query_len, void* workspace, int64_t workspace_bytes, int dtype, void* stream) {
  if (rows == 0 || num_seqs == 0) return 0;
  LV_CHECK(heads > 0 && kv_heads > 0 && heads % kv_heads == 0, "heads must be a multiple of kv_heads");
  LV_CHECK(kpad % 8 == 0 && vpad > 0 && vdim > 0 && vdim <= vpad && kpad <= 8192 && vpad <= 8192,
           "key rows are multiples of 8 elements, value rows at least vdim");
  LV_CHECK(max_blocks > 0 && num_blocks > 0 && block_size > 0, "an empty cache");
  LV_CHECK(num_seqs <= 65535 && heads <= 65535 && max_query_len > 0, "too many sequences or heads, or no query");
  HeadAttnParams p{};
  p.out = out; p.out_stride = out_stride; p.q = q; p.k_cache = key_cache; p.v_cache = value_cache;
  p.gate = gate; p.gate_stride = gate_stride; p.block_tables = block_tables; p.seq_lens = seq_lens;
  p.query_start_loc = query_start_loc; p.num_seqs = num_seqs; p.rows = rows; p.heads = heads; p.kv_heads = kv_heads;
  p.kpad = kpad; p.vpad = vpad; p.vdim = vdim; p.max_blocks = max_blocks; p.block_size = block_size;
  p.max_block = (int)(num_blocks - 1); p.scale = scale; p.out_scale = out_scale;
  p.k_block_stride = k_block_stride; p.v_block_stride = v_block_stride;
  p.max_query_len = max_query_len; p.max_seq_len = max_seq_len; p.nsplit = 1;
  p.window = window; p.min_query_len = min_query_len;
  hipStream_t s = (hipStream_t)stream;
  if (takes_mfma(kpad, vpad, block_size, dtype)) {
    p.nsplit = decode_shares(rows, num_seqs, heads, kv_heads, max_seq_len);
    if (p.nsplit > 1) {
      LV_CHECK(workspace != nullptr && workspace_bytes >= (int64_t)rows * heads * p.nsplit * (vpad + 2) * 4,
               "workspace too small (see lvllm_head_attention_workspace_bytes)");
      p.part_o = (float*)workspace;
      p.part_ml = p.part_o + (int64_t)rows * heads * p.nsplit * vpad;
    }
    if (min_query_len <= kDecodeCols)  // (longer ones all take the chunk body)
      if (int rc = launch_head_decode(p, s)) return rc;
    if (max_query_len > 1)
      if (int rc = launch_head_prefill(p, s)) return rc;
    return 0;
  }
  LV_DISPATCH_DTYPE(dtype, {
    hipLaunchKernelGGL((head_attention_simple_kernel<scalar_t>), dim3(rows, heads), dim3(256),
                       (size_t)(kpad + 256 + vpad) * 4, s, p);
  });
  LV_LAUNCH_CHECK();
  return 0;
}
