// Paged attention with unequal key and value sizes: the dispatcher and the body for 32-bit elements and for sizes outside
// the MFMA bodies (see head_attention.h for the layouts).
#include <float.h>

#include <algorithm>

#include "head_attention.h"

namespace lvllm {

// One workgroup per (row, head): 256 keys per round, one per thread for the scores, then one value column per thread; the maps
// one after the other.
template <typename T>
__global__ __launch_bounds__(256) void head_attention_simple_kernel(const HeadAttnParams p) {
  using S = typename T::store_t;
  constexpr int x = 16 / sizeof(S);
  extern __shared__ float sm[];
  const int mpad = p.kpad / p.maps;
  float* sq = sm;               // [mpad]
  float* sp = sq + mpad;        // [256]
  float* sacc = sp + 256;       // [maps][vpad]
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
  const int bs = p.block_size;
  const int low = first_seen(p, n_keys - 1), kept = min(p.keep_first, low);
  const int seen = kept + n_keys - low;  // keys 0 .. kept - 1, low .. n_keys - 1
  auto key_of = [&](int i) { return i < kept ? i : i - kept + low; };
  auto block_of = [&](int key) { return (int64_t)min(max(table[min(key / bs, p.max_blocks - 1)], 0), p.max_block); };
  float f = 1.f;
  for (int map = 0; map < p.maps; ++map) {
    const S* q = (const S*)p.q + (((int64_t)row * p.heads + head) * p.maps + map) * mpad;
    float* acc_map = sacc + map * p.vpad;
    __syncthreads();
    for (int d = threadIdx.x; d < mpad; d += 256) sq[d] = T::to_float(q[d]);
    for (int d = threadIdx.x; d < p.vpad; d += 256) acc_map[d] = 0.f;
    float m = -FLT_MAX, l = 0.f;
    for (int i0 = 0; i0 < seen; i0 += 256) {
      __syncthreads();
      const int i = i0 + threadIdx.x;
      float score = -FLT_MAX;
      if (i < seen) {
        const int key = key_of(i);
        const S* kc = (const S*)p.k_cache + block_of(key) * p.k_block_stride +
                      ((int64_t)kvh * p.kpad + map * mpad) * bs + (key % bs) * x;
        float acc = 0.f;
        for (int d = 0; d < mpad; d += x) {
          const Vec16<T> kv = *reinterpret_cast<const Vec16<T>*>(kc + (int64_t)(d / x) * bs * x);
#pragma unroll
          for (int j = 0; j < x; ++j) acc = fmaf(sq[d + j], T::to_float(kv.v[j]), acc);
        }
        score = acc * p.scale;
        if (p.softcap > 0.f) score = p.softcap * tanhf(score / p.softcap);
      }
      float mx = wave_max(score);
      if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = mx;
      __syncthreads();
      const float m_new = fmaxf(m, fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3])));
      const float corr = expf(m - m_new);
      const float e = i < seen ? expf(score - m_new) : 0.f;
      sp[threadIdx.x] = e;
      __syncthreads();
      l = l * corr + block_sum(e, red);
      m = m_new;
      const int nk = min(256, seen - i0);
      for (int d = threadIdx.x; d < p.vpad; d += 256) {
        float acc = acc_map[d] * corr;
        for (int j = 0; j < nk; ++j) {
          const int key = key_of(i0 + j);
          const S* vc = (const S*)p.v_cache + block_of(key) * p.v_block_stride + ((int64_t)kvh * p.vpad + d) * bs + key % bs;
          acc = fmaf(sp[j], T::to_float(*vc), acc);
        }
        acc_map[d] = acc;
      }
    }
    if (p.sink != nullptr) l += expf(p.sink[head] - m);
    if (p.maps == 1) {
      f = 1.f / l;
    } else {  // (a thread's columns are its own)
      const float w = (map == 0 ? 1.f : -p.map_weight) / l;
      for (int d = threadIdx.x; d < p.vpad; d += 256) {
        acc_map[d] *= w;
        if (map == 1) sacc[d] += acc_map[d];
      }
    }
  }
  if (p.maps == 2) {
    float ss = 0.f;
    for (int d = threadIdx.x; d < p.vdim; d += 256) ss = fmaf(sacc[d], sacc[d], ss);
    f = 1.f / sqrtf(block_sum(ss, red) / (float)p.vdim + p.map_eps);
  }
  f *= gate_of<T>(p, row, head);
  for (int d = threadIdx.x; d < p.vdim; d += 256) out[d] = T::from_float(sacc[d] * f);
}

}  // namespace lvllm

using namespace lvllm;

static bool mfma_size(int n, int least) {
  return n == least || n == 64 || n == 96 || n == 128 || n == 192 || n == 256;
}

static bool takes_mfma(int kpad, int vpad, int maps, int block_size, int dtype) {
  return dtype == LVLLM_BF16 && block_size == 16 && mfma_size(kpad, 64) && !(maps == 2 && kpad == 96) && mfma_size(vpad, 32);
}

// Shares the keys of a sequence are cut into: enough workgroups to fill the chip, none of under 256 keys, and none at all
// beside large prompt portions
static int decode_shares(int rows, int num_seqs, int heads, int kv_heads, int max_seq_len, const lvllm_head_options& o) {
  if (rows > 512) return 1;
  const int wgs = num_seqs * kv_heads * ((heads / kv_heads * o.maps + kDecodeCols - 1) / kDecodeCols);
  int n = (1024 + wgs - 1) / wgs;
  int64_t keys = max_seq_len;
  if (o.window > 0) keys = std::min<int64_t>(keys, (int64_t)o.window + o.keep_first + kDecodeCols);
  if (o.chunk > 0) keys = std::min<int64_t>(keys, (int64_t)o.chunk + o.keep_first + kDecodeCols);
  const int most = (int)((keys + 255) / 256);
  n = n < most ? n : most;
  return n < 1 ? 1 : n > 64 ? 64 : n;
}

static int64_t shares_bytes(int rows, int heads, int vpad, int maps, int n) {
  return maps > 1 || n > 1 ? (int64_t)rows * heads * maps * n * (vpad + 2) * 4 : 0;
}

extern "C" int64_t lvllm_head_attention_workspace_bytes(int rows, int num_seqs, int heads, int kv_heads, int kpad, int vpad,
                                                        int block_size, int max_seq_len, const lvllm_head_options* options,
                                                        int dtype) {
  const lvllm_head_options& o = *options;
  if (heads <= 0 || kv_heads <= 0 || rows <= 0 || num_seqs <= 0 || !takes_mfma(kpad, vpad, o.maps, block_size, dtype)) return 0;
  return shares_bytes(rows, heads, vpad, o.maps, decode_shares(rows, num_seqs, heads, kv_heads, max_seq_len, o));
}

extern "C" int lvllm_head_attention(void* out, int64_t out_stride, const void* q, const void* key_cache,
                                    const void* value_cache, const void* gate, int64_t gate_stride,
                                    const int32_t* block_tables, const int32_t* seq_lens, const int32_t* query_start_loc,
                                    int num_seqs, int rows, int heads, int kv_heads, int kpad, int vpad, int vdim,
                                    int max_blocks, int block_size, int64_t num_blocks, float scale, float out_scale,
                                    int64_t k_block_stride, int64_t v_block_stride, int max_query_len, int max_seq_len,
                                    const lvllm_head_options* options, void* workspace, int64_t workspace_bytes, int dtype,
                                    void* stream) {
  if (rows == 0 || num_seqs == 0) return 0;
  const lvllm_head_options& o = *options;
  LV_CHECK(heads > 0 && kv_heads > 0 && heads % kv_heads == 0, "heads must be a multiple of kv_heads");
  LV_CHECK(o.maps == 1 || o.maps == 2, "one or two maps");
  LV_CHECK(kpad % (8 * o.maps) == 0 && vpad > 0 && vdim > 0 && vdim <= vpad && kpad <= 8192 && vpad <= 4096,
           "key rows are multiples of 8 elements, value rows at least vdim");
  LV_CHECK(max_blocks > 0 && num_blocks > 0 && block_size > 0, "an empty cache");
  LV_CHECK(num_seqs <= 65535 && heads <= 65535 && max_query_len > 0, "too many sequences or heads, or no query");
  LV_CHECK(o.keep_first >= 0 && o.softcap >= 0.f, "negative option");
  HeadAttnParams p{};
  p.out = out; p.out_stride = out_stride; p.q = q; p.k_cache = key_cache; p.v_cache = value_cache;
  p.gate = gate; p.gate_stride = gate_stride; p.block_tables = block_tables; p.seq_lens = seq_lens;
  p.query_start_loc = query_start_loc; p.num_seqs = num_seqs; p.rows = rows; p.heads = heads; p.kv_heads = kv_heads;
  p.kpad = kpad; p.vpad = vpad; p.vdim = vdim; p.max_blocks = max_blocks; p.block_size = block_size;
  p.max_block = (int)(num_blocks - 1); p.scale = scale; p.out_scale = out_scale;
  p.k_block_stride = k_block_stride; p.v_block_stride = v_block_stride;
  p.max_query_len = max_query_len; p.max_seq_len = max_seq_len; p.nsplit = 1;
  p.window = o.window; p.chunk = o.chunk; p.keep_first = o.keep_first; p.maps = o.maps; p.min_query_len = o.min_query_len;
  p.softcap = o.softcap; p.sink = o.sink; p.map_weight = o.map_weight; p.map_eps = o.map_eps;
  hipStream_t s = (hipStream_t)stream;
  if (takes_mfma(kpad, vpad, o.maps, block_size, dtype)) {
    p.nsplit = decode_shares(rows, num_seqs, heads, kv_heads, max_seq_len, o);
    if (const int64_t need = shares_bytes(rows, heads, vpad, o.maps, p.nsplit)) {
      LV_CHECK(workspace != nullptr && workspace_bytes >= need, "workspace too small (see lvllm_head_attention_workspace_bytes)");
      p.part_o = (float*)workspace;
      p.part_ml = p.part_o + (int64_t)rows * heads * o.maps * p.nsplit * vpad;
    }
    if (o.min_query_len <= kDecodeCols)  // (longer ones all take the chunk body)
      if (int rc = o.maps == 2 ? launch_head_decode_maps(p, s) : launch_head_decode(p, s)) return rc;
    if (max_query_len > 1)
      if (int rc = o.maps == 2 ? launch_head_prefill_maps(p, s) : launch_head_prefill(p, s)) return rc;
    return 0;
  }
  const size_t smem = (size_t)(kpad / o.maps + 256 + o.maps * vpad) * 4;
  LV_DISPATCH_DTYPE(dtype, {
    if (smem > 64 * 1024)
      (void)hipFuncSetAttribute((const void*)head_attention_simple_kernel<scalar_t>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)smem);
    hipLaunchKernelGGL((head_attention_simple_kernel<scalar_t>), dim3(rows, heads), dim3(256), smem, s, p);
  });
  LV_LAUNCH_CHECK();
  return 0;
}
