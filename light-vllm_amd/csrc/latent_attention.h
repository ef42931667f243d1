// Latent attention for gfx950: a layer caches, per token, one latent c (kv_rank numbers) and one rotated key part (rot_dim
// numbers) that all heads share; head h's key is [U_h c | k_rot] and its value V_h c.  A query sees the keys of the last
// `window` positions, itself included (window <= 0: all of them).
//
// Two ways through, the same sums in another order:
//   * absorbed: the query is taken into latent space once, q' = [U_h^T q | q_rot], scores and weighted sums run on the cached
//     rows themselves (all heads on one row: bound by the cache's bytes), and V_h is applied to the summed latents.  Single
//     tokens and portions of up to `absorbed_max` tokens;
//   * expanded: the window's latents are gathered, keys and values of all heads made by one library product, and
//     head_attention runs over them.  Longer portions.
//
// sink[h], where given, is one more score of head h's softmax, without a key.
//
//   cache  [num_blocks, block_size, cpad + rpad]: c, zeros to cpad, the rotated part, zeros to the row's end
//   q'     [rows, heads, cpad + rpad], the same row layout
// Scores, softmax and accumulation are fp32.
#pragma once
#include "rotation.h"

namespace lvllm {

struct LatentAttnParams {
  void* out;               // row r, head h at r * out_stride + h * vdim
  const void *q, *cache;
  const void *uv, *gate;   // [heads, vpad, cpad], zero-padded; gate [rows, heads] (gate_stride apart) or null
  const float* sink;       // [heads] or null
  const int32_t *block_tables, *seq_lens, *query_start_loc;
  float *part_o, *part_ml;  // shares: [rows, heads, nsplit, cpad] and [rows, heads, nsplit, 2]
  int num_seqs, rows, heads, cpad, rpad, max_blocks, block_size, max_block, nsplit, window, absorbed_max, max_query_len;
  int vdim, vpad;
  float scale;
  int64_t block_stride, out_stride, gate_stride;
};

bool latent_takes_mfma(int cpad, int rpad, int block_size, int dtype);
int launch_latent_mfma(const LatentAttnParams& p, hipStream_t s);

// The first key position `pos` sees.
__device__ __forceinline__ int first_key(int pos, int window) { return window > 0 ? max(0, pos - window + 1) : 0; }

}  // namespace lvllm
