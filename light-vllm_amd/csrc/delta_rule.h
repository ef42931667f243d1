// Gated delta rule for gfx950: a matrix state S [dk, dv] per head, one decay per key channel, and a write that replaces what the
// state returns for the token's key:
//
//     S <- diag(g_t) S;   u_t = beta_t (v_t - S^T k_t);   S <- S + k_t u_t^T;   o_t = S^T q_t
//     out = o / rms(o) * norm_weight * sigmoid(gate)                            (per head)
//
// q, k and v come out of short convolutions (short_conv.h); q and k are then made unit vectors (x / sqrt(sum x^2 + 1e-6)), q
// times dk^-1/2 besides.  `heads / kv_heads` neighbouring heads share a q and a k.  ln g = -scale * softplus(A u + bias) per head
// and channel (log_decay.h), beta = sigmoid of one logit per head, gate = B z per head and value entry; A and B have a low rank.
//
// Two bodies:
//   * steps of single tokens: ONE launch per mixer, a workgroup per (head, sequence): convolutions, unit norms, both low-rank
//     products, state update, read-out, norm and gate.  With w = diag(g) S the read-out is w^T q + (k . q) u, so both products
//     with the state take one pass and one reduction; the state stays in registers between the pass and the update;
//   * portions, in chunks of 16 tokens.  With G_t the product of a chunk's decays up to token t, the u of a chunk solve the unit
//     lower triangular system
//         u_t + beta_t sum_{i < t} [k_t . (G_t / G_i) k_i] u_i = beta_t (v_t - (G_t k_t)^T S_0)
//     - delta_prepare_kernel, all chunks at once: the system's matrix on fp32 MFMAs, and its solution by substitution for both
//       right sides, U = solve(beta v) and W = solve(beta G k), beside the masked q . k products, q from the chunk's start and
//       k to its end;
//     - delta_scan_kernel, chunk after chunk: u = U - W S,  o = (G q)^T S + P u,  S <- G_end S + (k to the end)^T u.  The state's
//       columns are independent: a workgroup takes 16 NV of them, its four waves a quarter of the key channels each.  What it
//       reads is in fragment order and asked for several chunks ahead;
//     - head_norm_gate.h.
//
// Everything but the projections' results, the convolutions' and the gate is fp32.  Rows, sequences and slots as in recurrent.h.
#pragma once
#include "log_decay.h"
#include "short_conv.h"

namespace lvllm {

constexpr float kUnitEps = 1e-6f;

struct DeltaStepParams {
  void* out;               // row r, head h at r * out_stride + h * dv
  const void* x;           // rows before the convolution, x_stride apart: q at 0, k at k_at, v at v_at
  const void *u, *z, *beta;  // low-rank inputs of decay and gate, logits of beta; x_stride apart
  const float* conv_weight;  // [taps, channels]
  float* conv_state;
  const void *decay_w, *gate_w;  // [rank in pieces of 16 bytes][heads * dk (dv)][one piece]
  const float *decay_scale, *decay_bias, *norm_weight;  // [heads * dk], [heads * dk], [dv]
  float* state;
  const int32_t *state_slots, *seq_lens;
  int64_t out_stride, x_stride, conv_stride, state_stride;
  int k_at, v_at, taps, channels, decay_rank, gate_rank, num_seqs, num_slots, heads, kv_heads, dk, dv;
  float q_scale, eps;
};

// Pieces of one (chunk, head) in the workspace, in floats.  W, q and k: 16-byte piece `lane` of a tile of 16 key channels (W, q:
// row lane % 16, channels 4 (lane / 16) ..; k: channel lane % 16, rows 4 (lane / 16) ..).  U, per tile of 16 value columns, and P:
// four runs of 64, entry `lane` of run r being row 4 (lane / 16) + r, column lane % 16 (P: row lane % 16, column
// 4 (lane / 16) + r).
struct ChunkLayout {
  int dkp, dvp;  // multiples of 64 and 16
  __host__ __device__ __forceinline__ int w() const { return 0; }
  __host__ __device__ __forceinline__ int q() const { return 16 * dkp; }
  __host__ __device__ __forceinline__ int k() const { return 32 * dkp; }
  __host__ __device__ __forceinline__ int u() const { return 48 * dkp; }
  __host__ __device__ __forceinline__ int p() const { return 48 * dkp + 16 * dvp; }
  __host__ __device__ __forceinline__ int end() const { return 48 * dkp + 16 * dvp + 256; }
  __host__ __device__ __forceinline__ int size() const { return 49 * dkp + 16 * dvp + 256; }
};

struct DeltaChunkParams {
  const void *y, *beta;    // rows behind the convolution: q at 0, k at k_at, v at v_at; logits of beta
  const float* log_decay;  // [rows, heads, dk]
  float *chunks, *o;       // [chunk slots, heads, layout.size()], [rows, heads, dv]
  float* state;
  const int32_t *state_slots, *query_start_loc, *seq_lens;
  int64_t y_stride, beta_stride, state_stride;
  ChunkLayout layout;
  int k_at, v_at, num_seqs, num_slots, heads, kv_heads, dk, dv;
  float q_scale;
};

// Chunk i of sequence s has slot query_start_loc[s] / 16 + s + i: unique, and below rows / 16 + num_seqs
__device__ __forceinline__ int chunk_slot_base(const int32_t* query_start_loc, int s) { return query_start_loc[s] / kChunk + s; }

}  // namespace lvllm
