// Linear recurrences with a matrix state per head and one decay per key channel, for gfx950:
//
//     S_t = diag(w_t) S_{t-1} + k_t v_t^T          S [dk, dv], fp32, carried per sequence
//     o_t = S_t^T q_t                              (plain read-out), or
//     o_t = (S_{t-1} + diag(u) k_t v_t^T)^T q_t    (bonus read-out: u weighs the current token)
//
// and the low-rank data-dependent decays that drive them:
//
//     z = A f(u_t) + bias,   ln w = logsigmoid(z) / tau   (f = identity)   or   ln w = -exp(z)   (f = tanh)
//
// Two bodies:
//   * steps of single tokens (decode): ONE launch per mixer -- decay, state update, read-out, per-head RMS norm and gate --
//     a workgroup per (sequence, head) that streams the head's state through registers once: HBM-bound;
//   * everything else: the decays of all heads as one fp32-MFMA product, then chunks of 16 tokens on fp32 MFMAs
//     (chunk_mix_kernel): per chunk the decay from its start is folded into q, the decay to its end into k; the masked
//     16 x 16 products inside the chunk, the read-out of the state before it and the state update are matrix products, the
//     per-head norm and gate its epilogue.  State tiles are MFMA accumulators AND, without a move, the B operands of the
//     read-out (k-step r of a tile contracts rows {r, 4 + r, 8 + r, 12 + r}: accumulator register r of every lane).
//     Sequences too few to fill the chip are cut into segments of chunks, whose states are found first.
//   Inside a chunk the decay between two tokens is the product of two factors measured from the chunk's middle; channels
//   that decay too fast for that (a factor would leave fp32's range) are left out and added pair by pair.
//
// Everything but the projections' results (q, k, v, the low-rank input) is fp32: decays and their logarithms, the state,
// the read-out.  Rows are the new tokens of `num_seqs` sequences back to back (query_start_loc); a sequence whose tokens
// are all in this step (seq_lens == its rows) starts from a zero state, every other one from its slot.
#include "common.h"

namespace lvllm {

enum { kDecayLogSigmoid = 0, kDecayNegExp = 1 };

// e^x, |x| up to a few hundred: 2^(x log2 e) with the product's rounding error put back
__device__ __forceinline__ float exp_of(float x) {
  const float t = x * 1.44269502e+0f;
  const float lo = fmaf(x, 1.44269502e+0f, -t) + x * 1.92596299e-8f;
  const float r = __builtin_amdgcn_exp2f(t);
  return fmaf(r, lo * 0.693147182f, r);
}

__device__ __forceinline__ float log_decay_of(float z, int kind, float inv_tau) {
  if (kind == kDecayNegExp) return -exp_of(fminf(z, 9.f));  // (exp(-exp(9)) is 0: a finite logarithm keeps sums finite)
  return (fminf(z, 0.f) - log1pf(exp_of(-fabsf(z)))) * inv_tau;
}

typedef float r_f32x4_t __attribute__((ext_vector_type(4)));
__device__ __forceinline__ r_f32x4_t mfma_f32(float a, float b, r_f32x4_t c) {
  return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0);
}

// ---- ln w [rows, channels] ---------------------------------------------------------------------------------------
// A workgroup per 64 rows x 128 channels; f(u) through LDS, a wave's two tiles of 16 channels against all four row tiles.
constexpr int kDecayRows = 64, kDecayCols = 128;
template <typename T>
__global__ __launch_bounds__(256) void log_decay_kernel(float* __restrict__ out, const typename T::store_t* __restrict__ u,
                                                        const int64_t u_stride, const float* __restrict__ a_t,  // [rank, channels]
                                                        const float* __restrict__ bias, const int kind,
                                                        const float inv_tau, const int rows, const int rank,
                                                        const int channels) {
  extern __shared__ float su[];  // [kDecayRows][ld]
  const int rank4 = (rank + 3) & ~3, ld = rank4 + 1;
  const int row0 = blockIdx.y * kDecayRows, nr = min(kDecayRows, rows - row0);
  for (int k = threadIdx.x & 63; k < rank4; k += 64) {
    constexpr int N = kDecayRows / 4;
    const int r0 = threadIdx.x >> 6;
    typename T::store_t raw[N];  // (all of a thread's loads in flight at once)
#pragma unroll
    for (int i = 0; i < N; ++i) raw[i] = u[(int64_t)(row0 + min(r0 + 4 * i, nr - 1)) * u_stride + min(k, rank - 1)];
#pragma unroll
    for (int i = 0; i < N; ++i) {
      const float f = k < rank ? T::to_float(raw[i]) : 0.f;
      su[(r0 + 4 * i) * ld + k] = kind == kDecayNegExp ? tanhf(f) : f;
    }
  }
  __syncthreads();
  const int lane = threadIdx.x & 63, g = lane >> 4, c = lane & 15;
  const int ch0 = blockIdx.x * kDecayCols + __builtin_amdgcn_readfirstlane(threadIdx.x >> 6) * 32 + c;
  const float* b0 = a_t + min(ch0, channels - 1);
  const float* b1 = a_t + min(ch0 + 16, channels - 1);
  r_f32x4_t z[2][4];
#pragma unroll
  for (int j = 0; j < 2; ++j)
#pragma unroll
    for (int i = 0; i < 4; ++i) z[j][i] = r_f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll 8
  for (int k0 = 0; k0 < rank4; k0 += 4) {
    const int64_t at = (int64_t)min(k0 + g, rank - 1) * channels;  // (beyond the rank: f(u) is zero)
    const float x0 = b0[at], x1 = b1[at];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const float a = su[(16 * i + c) * ld + k0 + g];
      z[0][i] = mfma_f32(a, x0, z[0][i]);
      z[1][i] = mfma_f32(a, x1, z[1][i]);
    }
  }
#pragma unroll
  for (int j = 0; j < 2; ++j) {
    const int ch = ch0 + 16 * j;
    if (ch >= channels) continue;
    const float bb = bias[ch];
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int row = 16 * i + 4 * g + r;
        if (row < nr) out[(int64_t)(row0 + row) * channels + ch] = log_decay_of(z[j][i][r] + bb, kind, inv_tau);
      }
  }
}

// ---- token-by-token scan -----------------------------------------------------------------------------------------
// One workgroup per (sequence, head, 64 value columns): wave w holds state rows [w * NR, w * NR + NR) of its 64 columns
// in registers, tokens come in tiles of kScanTile through LDS, the four waves' partial read-outs meet in LDS per tile.
struct ScanParams {
  float* o;                        // [rows, heads, dv]
  const void *q, *k, *v;           // row r, head h at r * stride + h * dk (dv)
  int64_t q_stride, k_stride, v_stride;
  const float* log_decay;          // [rows, heads, dk]
  const float* bonus;              // [heads, dk] or null
  float q_scale;
  float* state;                    // [slots, heads, dk, dv], slots state_stride apart
  int64_t state_stride;
  const int32_t *state_slots, *query_start_loc, *seq_lens;
  int num_slots, heads, dk, dv;
};

constexpr int kScanTile = 16;

template <typename T, int NR>
__global__ __launch_bounds__(256) void scan_kernel(const ScanParams p) {
  using S = typename T::store_t;
  extern __shared__ float sm[];
  constexpr int DK = 4 * NR;
  float* sq = sm;                          // [tile][DK]
  float* sk = sq + kScanTile * DK;         // [tile][DK]
  float* sw = sk + kScanTile * DK;         // [tile][DK]
  float* sv = sw + kScanTile * DK;         // [tile][64]
  float* so = sv + kScanTile * 64;         // [4][tile][64]
  float* sb = so + 4 * kScanTile * 64;     // [DK]
  const int head = blockIdx.x, v0 = blockIdx.y * 64, seq = blockIdx.z;
  const int lane = threadIdx.x & 63;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int qbeg = p.query_start_loc[seq], qlen = p.query_start_loc[seq + 1] - qbeg;
  if (qlen <= 0) return;
  const int slot = p.state_slots[seq];
  const bool live = slot >= 0 && slot < p.num_slots;
  const int col = v0 + lane;
  const bool col_ok = col < p.dv;
  float* st = p.state + (int64_t)(live ? slot : 0) * p.state_stride + (int64_t)head * p.dk * p.dv + col;
  const bool fresh = p.seq_lens[seq] <= qlen || !live;
  float s[NR];
#pragma unroll
  for (int i = 0; i < NR; ++i) {
    const int r = wave * NR + i;
    s[i] = (!fresh && col_ok && r < p.dk) ? st[(int64_t)r * p.dv] : 0.f;
  }
  const bool has_bonus = p.bonus != nullptr;
  for (int i = threadIdx.x; i < DK; i += 256) sb[i] = (has_bonus && i < p.dk) ? p.bonus[head * p.dk + i] : 0.f;

  for (int t0 = 0; t0 < qlen; t0 += kScanTile) {
    const int nt = min(kScanTile, qlen - t0);
    __syncthreads();
    for (int i = threadIdx.x; i < kScanTile * DK; i += 256) {
      const int t = i / DK, d = i - t * DK;
      const bool ok = t < nt && d < p.dk;
      const int64_t row = qbeg + t0 + t;
      sq[i] = ok ? T::to_float(((const S*)p.q)[row * p.q_stride + head * p.dk + d]) * p.q_scale : 0.f;
      sk[i] = ok ? T::to_float(((const S*)p.k)[row * p.k_stride + head * p.dk + d]) : 0.f;
      sw[i] = ok ? expf(p.log_decay[(row * p.heads + head) * p.dk + d]) : 1.f;
    }
    for (int i = threadIdx.x; i < kScanTile * 64; i += 256) {
      const int t = i >> 6, d = v0 + (i & 63);
      sv[i] = (t < nt && d < p.dv) ? T::to_float(((const S*)p.v)[(qbeg + t0 + t) * p.v_stride + head * p.dv + d]) : 0.f;
    }
    __syncthreads();
    for (int t = 0; t < nt; ++t) {
      const float vv = sv[t * 64 + lane];
      const float* q = sq + t * DK + wave * NR;
      const float* k = sk + t * DK + wave * NR;
      const float* w = sw + t * DK + wave * NR;
      float acc = 0.f;
      if (has_bonus) {
        const float* u = sb + wave * NR;
#pragma unroll
        for (int i = 0; i < NR; ++i) {
          const float kv = k[i] * vv;
          acc = fmaf(q[i], fmaf(u[i], kv, s[i]), acc);
          s[i] = fmaf(w[i], s[i], kv);
        }
      } else {
#pragma unroll
        for (int i = 0; i < NR; ++i) {
          s[i] = fmaf(w[i], s[i], k[i] * vv);
          acc = fmaf(q[i], s[i], acc);
        }
      }
      so[(wave * kScanTile + t) * 64 + lane] = acc;
    }
    __syncthreads();
    for (int i = threadIdx.x; i < nt * 64; i += 256) {
      const int t = i >> 6, d = v0 + (i & 63);
      if (d < p.dv) {
        const float r = (so[i] + so[kScanTile * 64 + i]) + (so[2 * kScanTile * 64 + i] + so[3 * kScanTile * 64 + i]);
        p.o[((int64_t)(qbeg + t0 + t) * p.heads + head) * p.dv + d] = r;
      }
    }
  }
  if (live && col_ok) {
#pragma unroll
    for (int i = 0; i < NR; ++i) {
      const int r = wave * NR + i;
      if (r < p.dk) st[(int64_t)r * p.dv] = s[i];
    }
  }
}

template <typename T, int NR>
static int launch_scan(const ScanParams& p, int num_seqs, hipStream_t s) {
  const size_t smem = (size_t)(kScanTile * (3 * 4 * NR + 64 + 4 * 64) + 4 * NR) * sizeof(float);
  if (smem > 64 * 1024)
    (void)hipFuncSetAttribute((const void*)scan_kernel<T, NR>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)smem);
  hipLaunchKernelGGL((scan_kernel<T, NR>), dim3(p.heads, (p.dv + 63) / 64, num_seqs), dim3(256), smem, s, p);
  return 0;
}


// ---- chunks of 16 tokens ------------------------------------------------------------------------------------------
constexpr int kChunk = 16;
constexpr float kMaxHalfDecay = 60.f;  // ln of the largest factor measured from the middle of a chunk

struct MixParams {
  const void *q, *k, *v;  // row r, head h at r * stride + h * dk (dv)
  int64_t q_stride, k_stride, v_stride;
  const void* u;          // low-rank input, row stride u_stride
  int64_t u_stride;
  const float* a_t;       // [rank, heads * dk]
  const float* decay_bias;
  int kind, rank;
  float inv_tau;
  const float* bonus;     // [heads, dk] or null
  float q_scale;
  float* state;
  int64_t state_stride;
  const int32_t *state_slots, *query_start_loc, *seq_lens;
  int num_seqs, num_slots, heads, dk, dv;
  // epilogue
  void* out;              // row r, head h at r * out_stride + h * dv
  int64_t out_stride;
  const void* gate;
  int64_t gate_stride;
  const float* norm_weight;
  int norm_head_stride;
  float eps, out_scale;
  bool vec_in, vec_out;   // rows of v and gate take 4-element loads, rows of `out` 4-element stores
  // chunked body
  const float* log_decay; // [rows, heads, dk]
  float* o;               // [rows, heads, dv], or null: the epilogue is applied where o is made
  int seg_chunks, max_segs;  // chunks per segment, segments of the longest sequence (1: not cut)
  float* seg_state;       // [segment slots, heads, dk, dv]
  float* seg_decay;       // [segment slots, heads, dkp]
};

// Segment k of sequence s has slot query_start_loc[s] / (tokens of a segment) + s + k: unique
__device__ __forceinline__ int seg_slot_base(const MixParams& p, int s) {
  return p.query_start_loc[s] / (kChunk * p.seg_chunks) + s;
}

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

__host__ __device__ constexpr int mix_smem_floats(int NT, int NV) {
  return 4 * kChunk * (64 * NT + 4) + 4 * 256 + 4 * kChunk + 5 * kChunk * (16 * NV + 4) + 4 * NT;
}

// N neighbouring elements as loaded
template <typename T, int N>
struct Packed {
  using S = typename T::store_t;
  static constexpr int W = sizeof(S) == 4 ? N : (N + 1) / 2;
  uint32_t w[W];
  // elements col .. of a row of n (beyond it the last one); `vec`: 4-element loads are aligned
  __device__ __forceinline__ void load(const S* row, int col, int n, bool vec) {
    if constexpr (N >= 4) {
      if (vec && col + N <= n) {
        constexpr int V = W * 4 / N;  // words per 4 elements
#pragma unroll
        for (int j = 0; j < N / 4; ++j) {
          if constexpr (V == 2) {
            const uint2 x = *reinterpret_cast<const uint2*>(row + col + 4 * j);
            w[2 * j] = x.x; w[2 * j + 1] = x.y;
          } else {
            const uint4 x = *reinterpret_cast<const uint4*>(row + col + 4 * j);
            w[4 * j] = x.x; w[4 * j + 1] = x.y; w[4 * j + 2] = x.z; w[4 * j + 3] = x.w;
          }
        }
        return;
      }
    }
#pragma unroll
    for (int j = 0; j < N; ++j) {
      const S x = row[min(col + j, n - 1)];
      if constexpr (sizeof(S) == 4) w[j] = __builtin_bit_cast(uint32_t, x);
      else w[j / 2] = j % 2 == 0 ? (uint32_t)x : w[j / 2] | ((uint32_t)x << 16);
    }
  }
  __device__ __forceinline__ float at(int j) const {
    if constexpr (sizeof(S) == 4) return __builtin_bit_cast(float, w[j]);
    else return T::to_float((uint16_t)(w[j / 2] >> (16 * (j & 1))));
  }
};

// One workgroup per (sequence, head, slice of 16 * NV value columns, segment), walking its chunks in order.  Wave w owns key
// channels [w * 16 * NT, (w + 1) * 16 * NT): it scales q and k there, holds those rows of the state as accumulator tiles and
// forms partial in-chunk products and read-outs, which meet in LDS.  A lane loads channel c, tokens 4g .. 4g + 3 of a tile:
// scaled k is then the A operand of the state update as it is; q goes through LDS.
//   STATES: from a zero state, no read-out: a segment's last state and the product of its decays, of all segments but the
//   last.  Otherwise the segment's first state comes from the slot (sequences that are not cut) or from chunk_combine_kernel.
template <typename T, int NT, int NV, bool STATES>
__global__ __launch_bounds__(256, NT == 1 && NV <= 4 ? 3 : 2) void chunk_mix_kernel(const MixParams p) {
  using S = typename T::store_t;
  constexpr int DKP = 64 * NT;
  constexpr int LD = DKP + 4;       // row strides of the LDS images (bank spread of the 16-byte reads)
  constexpr int LO = 16 * NV + 4;
  extern __shared__ __attribute__((aligned(16))) float sm[];
  float* sq = sm;                   // [16][LD]: q from the middle of the chunk (fast decays: q)
  float* sk = sq + kChunk * LD;     // [16][LD]: k to the middle (fast decays: k)
  float* sr = sk + kChunk * LD;     // [16][LD]: q from the chunk's start
  float* sl = sr + kChunk * LD;     // [16][LD]: ln w (fast decays)
  float* spart = sl + kChunk * LD;  // [4 waves][16][16]: in-chunk products
  float* sdiag = spart + 4 * 256;   // [4 waves][16]: the bonus' diagonal
  float* so = sdiag + 4 * kChunk;   // [4 waves][16][LO]: read-outs
  float* sv = so + 4 * kChunk * LO; // [16][LO]: values
  int* swild = reinterpret_cast<int*>(sv + kChunk * LO);  // [4 NT]: channels of a tile that decay too fast for the factors
  const int head = blockIdx.x, v0 = blockIdx.y * 16 * NV;
  const bool cut = p.max_segs > 1;
  const int seq = cut ? blockIdx.z / p.max_segs : blockIdx.z, seg = cut ? blockIdx.z - seq * p.max_segs : 0;
  const int qbeg = p.query_start_loc[seq], qlen = p.query_start_loc[seq + 1] - qbeg;
  if (qlen <= 0) return;
  const int all_chunks = (qlen + kChunk - 1) / kChunk;
  const int first = cut ? seg * p.seg_chunks : 0;
  const int last = cut ? min(first + p.seg_chunks, all_chunks) : all_chunks;
  if (first >= all_chunks || (STATES && last == all_chunks)) return;
  const int lane = threadIdx.x & 63;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int g = lane >> 4, c = lane & 15;
  const int slot = p.state_slots[seq];
  const bool live = slot >= 0 && slot < p.num_slots;
  float* st = p.state + (int64_t)(live ? slot : 0) * p.state_stride + (int64_t)head * p.dk * p.dv;
  const int64_t seg_slot = cut ? seg_slot_base(p, seq) + seg : 0;
  float* seg_st = cut ? p.seg_state + (seg_slot * p.heads + head) * p.dk * p.dv : nullptr;
  const float* from = STATES ? nullptr : cut ? seg_st : (live && p.seq_lens[seq] > qlen) ? st : nullptr;
  r_f32x4_t s[NT][NV];
#pragma unroll
  for (int i = 0; i < NT; ++i)
#pragma unroll
    for (int j = 0; j < NV; ++j)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int row = (wave * NT + i) * 16 + 4 * g + r, col = v0 + 16 * j + c;
        s[i][j][r] = (from != nullptr && row < p.dk && col < p.dv) ? from[(int64_t)row * p.dv + col] : 0.f;
      }
  const bool has_bonus = p.bonus != nullptr;
  float bon[NT], prod[NT];
#pragma unroll
  for (int i = 0; i < NT; ++i) {
    const int ch = (wave * NT + i) * 16 + c;
    bon[i] = (has_bonus && ch < p.dk) ? p.bonus[head * p.dk + ch] : 0.f;
    prod[i] = 1.f;
  }
  // epilogue of this thread: token threadIdx.x / 16 of a chunk, NV columns from d0
  const int et = threadIdx.x >> 4, d0 = v0 + (threadIdx.x & 15) * NV;
  const bool epilogue = !STATES && p.o == nullptr;
  float nw[NV];
  if constexpr (!STATES) {
#pragma unroll
    for (int j = 0; j < NV; ++j)
      nw[j] = (epilogue && d0 + j < p.dv) ? p.norm_weight[head * p.norm_head_stride + d0 + j] * p.out_scale : 0.f;
  }

  struct Frag {
    S q[NT][4], k[NT][4];
    float l[NT][4];
    S v[STATES ? NV : 1][4];       // (STATES) tokens 4g .. 4g + 3 of column c of each tile
    Packed<T, NV> vrow, gate;      // else: this thread's NV columns of token et
  };
  // addresses are clamped to the sequence's rows and the head's columns; what lies beyond is masked when it is used
  auto load = [&](int ci, Frag& f) __attribute__((always_inline)) {
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int64_t row = qbeg + min(ci * kChunk + 4 * g + r, qlen - 1);
#pragma unroll
      for (int i = 0; i < NT; ++i) {
        const int ch = head * p.dk + min((wave * NT + i) * 16 + c, p.dk - 1);
        if constexpr (!STATES) f.q[i][r] = ((const S*)p.q)[row * p.q_stride + ch];
        f.k[i][r] = ((const S*)p.k)[row * p.k_stride + ch];
        f.l[i][r] = p.log_decay[row * p.heads * p.dk + ch];
      }
      if constexpr (STATES) {
#pragma unroll
        for (int j = 0; j < NV; ++j)
          f.v[j][r] = ((const S*)p.v)[row * p.v_stride + head * p.dv + min(v0 + 16 * j + c, p.dv - 1)];
      }
    }
    if constexpr (!STATES) {
      const int64_t row = qbeg + min(ci * kChunk + et, qlen - 1);
      f.vrow.load((const S*)p.v + row * p.v_stride + head * p.dv, d0, p.dv, p.vec_in);
      if (epilogue) f.gate.load((const S*)p.gate + row * p.gate_stride + head * p.dv, d0, p.dv, p.vec_in);
    }
  };
  Frag f;
  load(first, f);
  for (int ci = first; ci < last; ++ci) {
    const int nt = min(kChunk, qlen - ci * kChunk);
    if constexpr (!STATES) {
      float* at = sv + et * LO + (d0 - v0);
#pragma unroll
      for (int j = 0; j < NV; ++j) at[j] = f.vrow.at(j);
    }
    float kd[NT][4], end[NT];  // k scaled to the chunk's end; the chunk's decay
    bool wild = false;
    float diag[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int i = 0; i < NT; ++i) {
      const int ch = (wave * NT + i) * 16 + c;
      float l[4], kv[4];
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const bool ok = 4 * g + r < nt && ch < p.dk;
        l[r] = ok ? f.l[i][r] : 0.f;
        kv[r] = ok ? T::to_float(f.k[i][r]) : 0.f;
      }
      const ChunkSums cs(l, g, c, has_bonus);
      end[i] = exp_of(cs.h1 + cs.h2);
      if constexpr (STATES) {
#pragma unroll
        for (int r = 0; r < 4; ++r) kd[i][r] = kv[r] * exp_of(cs.left[r]);
        prod[i] *= end[i];
      } else {
        const bool mild = -cs.h1 < kMaxHalfDecay && -cs.h2 < kMaxHalfDecay;
        wild = wild || !mild;
        const uint64_t fast_decays = __ballot(!mild);
        if (lane == 0) swild[wave * NT + i] = (int)(fast_decays & 0xffff);
        const float to_mid = exp_of(cs.h1), from_mid = exp_of(cs.h2);
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int t = 4 * g + r;
          const float qv = t < nt && ch < p.dk ? T::to_float(f.q[i][r]) * p.q_scale : 0.f;
          const float qh = mild ? qv * exp_of(cs.half_q[r]) : 0.f, kh = mild ? kv[r] * exp_of(cs.half_k[r]) : 0.f;
          sq[t * LD + ch] = qh;
          sk[t * LD + ch] = kh;
          float qs = qh * to_mid, ks = kh * from_mid;
          if (!mild) {
            qs = qv * exp_of(cs.read[r]);
            ks = kv[r] * exp_of(cs.left[r]);
          }
          sr[t * LD + ch] = qs;
          kd[i][r] = ks;
          diag[r] = fmaf(qv * bon[i], kv[r], diag[r]);
        }
      }
    }
    // the next chunk's loads are in flight during the products and the epilogue of this one
    const Packed<T, NV> gate = f.gate;
    S vraw[STATES ? NV : 1][4];
    if constexpr (STATES) {
#pragma unroll
      for (int j = 0; j < NV; ++j)
#pragma unroll
        for (int r = 0; r < 4; ++r) vraw[j][r] = f.v[j][r];
    }
    if (ci + 1 < last) load(ci + 1, f);
    float a = 0.f;  // A operand of the in-chunk part: row c, token 4g + wave
    if constexpr (!STATES) {
      if (has_bonus) {
#pragma unroll
        for (int r = 0; r < 4; ++r) {
#pragma unroll
          for (int m = 1; m < 16; m <<= 1) diag[r] += __shfl_xor(diag[r], m);
          if (c == 0) sdiag[wave * 16 + 4 * g + r] = diag[r];
        }
      }
      // this wave's channels only: what it wrote itself, no barrier needed
      __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
      __builtin_amdgcn_wave_barrier();
      r_f32x4_t a4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int i = 0; i < NT; ++i) {
        const int ch0 = (wave * NT + i) * 16 + 4 * g;
        const float4 qa = *reinterpret_cast<const float4*>(sq + c * LD + ch0);
        const float4 kb = *reinterpret_cast<const float4*>(sk + c * LD + ch0);
        a4 = mfma_f32(qa.x, kb.x, a4);
        a4 = mfma_f32(qa.y, kb.y, a4);
        a4 = mfma_f32(qa.z, kb.z, a4);
        a4 = mfma_f32(qa.w, kb.w, a4);
      }
#pragma unroll
      for (int r = 0; r < 4; ++r) spart[wave * 256 + (4 * g + r) * 16 + c] = a4[r];
      if (__syncthreads_or(wild)) {  // the products of the channels left out above, pair by pair
#pragma unroll
        for (int i = 0; i < NT; ++i) {
          const int ch = (wave * NT + i) * 16 + c;
          if (swild[wave * NT + i] >> c & 1) {
#pragma unroll
            for (int r = 0; r < 4; ++r) {
              const int t = 4 * g + r;
              const bool ok = t < nt && ch < p.dk;
              const int64_t row = qbeg + min(ci * kChunk + t, qlen - 1);
              const int col = head * p.dk + min(ch, p.dk - 1);
              sq[t * LD + ch] = ok ? T::to_float(((const S*)p.q)[row * p.q_stride + col]) * p.q_scale : 0.f;
              sk[t * LD + ch] = ok ? T::to_float(((const S*)p.k)[row * p.k_stride + col]) : 0.f;
              sl[t * LD + ch] = ok ? p.log_decay[row * p.heads * p.dk + col] : 0.f;
            }
          }
        }
        __syncthreads();
        const int ti = threadIdx.x >> 4, tj = threadIdx.x & 15;
        if (tj <= ti) {
          float sum = 0.f;
          for (int i = 0; i < 4 * NT; ++i) {
            for (int left = swild[i]; left != 0; left &= left - 1) {
              const int ch = i * 16 + __builtin_ctz(left);
              float between = 0.f;
              for (int t = tj + 1; t < (has_bonus ? ti : ti + 1); ++t) between += sl[t * LD + ch];
              sum = fmaf(sq[ti * LD + ch] * exp_of(between), sk[tj * LD + ch], sum);
            }
          }
          spart[threadIdx.x] += sum;
        }
        __syncthreads();
      }
      const int tj = 4 * g + wave, at = c * 16 + tj;
      if (has_bonus ? tj < c : tj <= c)
        a = (spart[at] + spart[256 + at]) + (spart[512 + at] + spart[768 + at]);
      else if (has_bonus && tj == c)
        a = (sdiag[c] + sdiag[16 + c]) + (sdiag[32 + c] + sdiag[48 + c]);
    }
    float4 qf[NT], e[NT];
#pragma unroll
    for (int i = 0; i < NT; ++i) {
      if constexpr (!STATES) qf[i] = *reinterpret_cast<const float4*>(sr + c * LD + (wave * NT + i) * 16 + 4 * g);
      e[i] = float4{__shfl(end[i], 4 * g), __shfl(end[i], 4 * g + 1), __shfl(end[i], 4 * g + 2), __shfl(end[i], 4 * g + 3)};
    }
#pragma unroll
    for (int j = 0; j < NV; ++j) {
      float v[4];
#pragma unroll
      for (int r = 0; r < 4; ++r) v[r] = STATES ? T::to_float(vraw[STATES ? j : 0][r]) : sv[(4 * g + r) * LO + 16 * j + c];
      if constexpr (!STATES) {
        r_f32x4_t o{0.f, 0.f, 0.f, 0.f};
        o = mfma_f32(a, wave == 0 ? v[0] : wave == 1 ? v[1] : wave == 2 ? v[2] : v[3], o);
#pragma unroll
        for (int i = 0; i < NT; ++i) {
          o = mfma_f32(qf[i].x, s[i][j][0], o);
          o = mfma_f32(qf[i].y, s[i][j][1], o);
          o = mfma_f32(qf[i].z, s[i][j][2], o);
          o = mfma_f32(qf[i].w, s[i][j][3], o);
        }
#pragma unroll
        for (int r = 0; r < 4; ++r) so[(wave * kChunk + 4 * g + r) * LO + 16 * j + c] = o[r];
      }
#pragma unroll
      for (int i = 0; i < NT; ++i) {
        r_f32x4_t n = s[i][j];
        n[0] *= e[i].x; n[1] *= e[i].y; n[2] *= e[i].z; n[3] *= e[i].w;
        n = mfma_f32(kd[i][0], v[0], n);
        n = mfma_f32(kd[i][1], v[1], n);
        n = mfma_f32(kd[i][2], v[2], n);
        n = mfma_f32(kd[i][3], v[3], n);
        s[i][j] = n;
      }
    }
    if constexpr (!STATES) {
      __syncthreads();  // (`so` is written again only behind the next chunk's first barrier)
      float o[NV], ss = 0.f;
#pragma unroll
      for (int j = 0; j < NV; ++j) {
        const float* at = so + et * LO + (d0 - v0) + j;
        o[j] = (at[0] + at[kChunk * LO]) + (at[2 * kChunk * LO] + at[3 * kChunk * LO]);
        if (d0 + j < p.dv) ss = fmaf(o[j], o[j], ss);
      }
      const int64_t row = qbeg + ci * kChunk + et;
      if (!epilogue) {
        if (et < nt)
#pragma unroll
          for (int j = 0; j < NV; ++j)
            if (d0 + j < p.dv) p.o[(row * p.heads + head) * p.dv + d0 + j] = o[j];
        continue;
      }
#pragma unroll
      for (int m = 8; m >= 1; m >>= 1) ss += __shfl_xor(ss, m);
      const float rms = 1.f / sqrtf(ss / p.dv + p.eps);
      if (et < nt) {
        S* out = (S*)p.out + row * p.out_stride + head * p.dv + d0;
#pragma unroll
        for (int j = 0; j < NV; ++j) {
          const float zg = gate.at(j);
          o[j] = o[j] * rms * nw[j] * (zg / (1.f + expf(-zg)));
        }
        if constexpr (NV >= 4) {
          if (p.vec_out && d0 + NV <= p.dv) {
#pragma unroll
            for (int j = 0; j < NV; j += 4) {
              const float w[4] = {o[j], o[j + 1], o[j + 2], o[j + 3]};
              store4<T>(out + j, w);
            }
            continue;
          }
        }
#pragma unroll
        for (int j = 0; j < NV; ++j)
          if (d0 + j < p.dv) out[j] = T::from_float(o[j]);
      }
    }
  }
  if (STATES && blockIdx.y == 0 && g == 0) {
#pragma unroll
    for (int i = 0; i < NT; ++i) p.seg_decay[(seg_slot * p.heads + head) * DKP + (wave * NT + i) * 16 + c] = prod[i];
  }
  if (STATES || (live && last == all_chunks)) {
    float* to = STATES ? seg_st : st;
#pragma unroll
    for (int i = 0; i < NT; ++i)
#pragma unroll
      for (int j = 0; j < NV; ++j)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int row = (wave * NT + i) * 16 + 4 * g + r, col = v0 + 16 * j + c;
          if (row < p.dk && col < p.dv) to[(int64_t)row * p.dv + col] = s[i][j][r];
        }
  }
}

// The first state of every segment, in place of the last state it would have had from zero: a thread per state element,
// sequential over the segments.
__global__ __launch_bounds__(256) void chunk_combine_kernel(const MixParams p, const int dkp) {
  const int head = blockIdx.y, seq = blockIdx.z;
  const int qlen = p.query_start_loc[seq + 1] - p.query_start_loc[seq];
  const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x, per_head = (int64_t)p.dk * p.dv;
  if (qlen <= 0 || i >= per_head) return;
  const int segs = (qlen + kChunk * p.seg_chunks - 1) / (kChunk * p.seg_chunks);
  const int slot = p.state_slots[seq];
  const bool live = slot >= 0 && slot < p.num_slots;
  float x = 0.f;
  if (live && p.seq_lens[seq] > qlen) x = p.state[(int64_t)slot * p.state_stride + head * per_head + i];
  const int64_t base = (int64_t)seg_slot_base(p, seq) * p.heads + head;
  float* st = p.seg_state + base * per_head + i;
  const float* de = p.seg_decay + base * dkp + i / p.dv;
  const int64_t st_step = p.heads * per_head, de_step = (int64_t)p.heads * dkp;
#pragma unroll 4
  for (int k = 0; k < segs - 1; ++k) {
    const float own = st[k * st_step], d = de[k * de_step];
    st[k * st_step] = x;
    x = fmaf(d, x, own);
  }
  st[(segs - 1) * st_step] = x;
}

// ---- single tokens -------------------------------------------------------------------------------------------------
// state that is not touched again before the next step: past the caches
__device__ __forceinline__ float4 load_stream(const float* p) {
  const r_f32x4_t v = __builtin_nontemporal_load(reinterpret_cast<const r_f32x4_t*>(p));
  return float4{v[0], v[1], v[2], v[3]};
}
__device__ __forceinline__ void store_stream(float* p, float4 v) {
  __builtin_nontemporal_store(r_f32x4_t{v.x, v.y, v.z, v.w}, reinterpret_cast<r_f32x4_t*>(p));
}

// One workgroup per (head, sequence), sequence s owning row s.  Thread (rg, cg): state columns 4 cg .. 4 cg + 3 of rows
// rg, rg + RG, ...  With PRE > 0 the thread's PRE state rows are loaded before anything else, so that the whole state is in
// flight while the decays are computed; PRE = 0 takes any size.
template <typename T, int PRE>
__global__ __launch_bounds__(256) void recurrent_decode_kernel(const MixParams p) {
  using S = typename T::store_t;
  extern __shared__ float sm[];
  const int head = blockIdx.x, seq = blockIdx.y, row = seq;
  const int dk = p.dk, dv = p.dv;
  const int slot = p.state_slots[seq];
  const bool live = slot >= 0 && slot < p.num_slots;
  const bool fresh = p.seq_lens[seq] <= 1 || !live;
  float* st = p.state + (int64_t)(live ? slot : 0) * p.state_stride + (int64_t)head * dk * dv;
  const bool vec = (dv & 3) == 0;
  const int cgs = vec ? dv / 4 : dv;           // column groups
  const int per = min(cgs, 256);               // threads along a row
  const int rgs = 256 / per;                   // row groups
  const int rg = threadIdx.x / per, cg0 = threadIdx.x - rg * per;
  // Loads return in order: the small operands go first, the state behind them, and both are in flight while the decays are
  // computed.  (dk <= 256: one key channel per thread; the first 256 values, low-rank inputs and columns likewise.)
  const int tid = threadIdx.x;
  const int kc = head * dk + min(tid, dk - 1), vc = head * dv + min(tid, dv - 1);
  const float u0 = T::to_float(((const S*)p.u)[(int64_t)row * p.u_stride + min(tid, p.rank - 1)]);
  const float q0 = T::to_float(((const S*)p.q)[(int64_t)row * p.q_stride + kc]) * p.q_scale;
  const float k0 = T::to_float(((const S*)p.k)[(int64_t)row * p.k_stride + kc]);
  const float v0 = T::to_float(((const S*)p.v)[(int64_t)row * p.v_stride + vc]);
  const float gate0 = T::to_float(((const S*)p.gate)[(int64_t)row * p.gate_stride + vc]);
  const float weight0 = p.norm_weight[head * p.norm_head_stride + min(tid, dv - 1)];
  const float bias0 = p.decay_bias[kc];
  const float bonus0 = p.bonus != nullptr ? p.bonus[kc] : 0.f;
  // z: the rank cut into parts, thread (part, channel)
  const int parts = 256 / dk, part_len = (p.rank + parts - 1) / parts;
  const int part = tid / dk, part_ch = tid - part * dk;
  const float* a = p.a_t + head * dk + part_ch;
  const int64_t a_step = (int64_t)p.heads * dk;
  constexpr int AR = PRE == 4 ? 16 : 32;
  float a_pre[AR];
#pragma unroll
  for (int i = 0; i < AR; ++i) a_pre[i] = a[min(part * part_len + i, p.rank - 1) * a_step];
  float4 pre[PRE > 0 ? PRE : 1];
  if constexpr (PRE > 0) {
#pragma unroll
    for (int i = 0; i < PRE; ++i) {
      pre[i] = float4{0.f, 0.f, 0.f, 0.f};
      const int r = rg + i * rgs;
      if (!fresh && rg < rgs && r < dk) pre[i] = load_stream(st + (int64_t)r * dv + 4 * cg0);
    }
  }
  float* sq = sm;            // [dk]
  float* sk = sq + dk;       // [dk]
  float* sw = sk + dk;       // [dk]
  float* su = sw + dk;       // [rank]
  float* sv = sm + ((3 * dk + p.rank + 3) & ~3);  // [dv], 16-byte aligned
  float* so = sv + dv;       // [row groups][dv]; before that the parts of z [256 / dk][dk]
  __shared__ float red[16];
  __shared__ float s_bonus;
  if (tid < p.rank) su[tid] = p.kind == kDecayNegExp ? tanhf(u0) : u0;
  for (int i = tid + 256; i < p.rank; i += 256) {
    const float f = T::to_float(((const S*)p.u)[(int64_t)row * p.u_stride + i]);
    su[i] = p.kind == kDecayNegExp ? tanhf(f) : f;
  }
  if (tid < dv) sv[tid] = v0;
  for (int i = tid + 256; i < dv; i += 256) sv[i] = T::to_float(((const S*)p.v)[(int64_t)row * p.v_stride + head * dv + i]);
  if (tid < dk) {
    sq[tid] = q0;
    sk[tid] = k0;
  }
  __syncthreads();
  if (part < parts) {
    const int r0 = part * part_len, r1 = min(r0 + part_len, p.rank);
    float z = 0.f;
#pragma unroll
    for (int i = 0; i < AR; ++i)
      if (r0 + i < r1) z = fmaf(su[r0 + i], a_pre[i], z);
    for (int r = r0 + AR; r < r1; ++r) z = fmaf(su[r], a[r * a_step], z);
    so[part * dk + part_ch] = z;
  }
  __syncthreads();
  float bsum = 0.f;
  if (tid < dk) {
    float z = bias0;
    for (int q = 0; q < parts; ++q) z += so[q * dk + tid];
    sw[tid] = expf(log_decay_of(z, p.kind, p.inv_tau));
    bsum = q0 * bonus0 * k0;
  }
  const bool has_bonus = p.bonus != nullptr;
  const float b = block_sum(bsum, red);  // (barriers: sw is visible behind it)
  if (threadIdx.x == 0) s_bonus = b;
  if constexpr (PRE > 0) {
    if (rg < rgs) {
      const float4 v = *reinterpret_cast<const float4*>(sv + 4 * cg0);
      float4 acc{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int i = 0; i < PRE; ++i) {
        const int r = rg + i * rgs;
        if (r < dk) {
          const float w = sw[r], k = sk[r], q = sq[r];
          const float4 s = pre[i];
          const float4 n{fmaf(w, s.x, k * v.x), fmaf(w, s.y, k * v.y), fmaf(w, s.z, k * v.z), fmaf(w, s.w, k * v.w)};
          const float4 rd = has_bonus ? s : n;
          acc.x = fmaf(q, rd.x, acc.x); acc.y = fmaf(q, rd.y, acc.y);
          acc.z = fmaf(q, rd.z, acc.z); acc.w = fmaf(q, rd.w, acc.w);
          if (live) store_stream(st + (int64_t)r * dv + 4 * cg0, n);
        }
      }
      *reinterpret_cast<float4*>(so + rg * dv + 4 * cg0) = acc;
    }
  } else if (rg < rgs) {
    for (int cg = cg0; cg < cgs; cg += per) {
      if (vec) {
        const float4 v = *reinterpret_cast<const float4*>(sv + 4 * cg);
        float4 acc{0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
        for (int r = rg; r < dk; r += rgs) {
          float4 s{0.f, 0.f, 0.f, 0.f};
          float* at = st + (int64_t)r * dv + 4 * cg;
          if (!fresh) s = *reinterpret_cast<const float4*>(at);
          const float w = sw[r], k = sk[r], q = sq[r];
          float4 n{fmaf(w, s.x, k * v.x), fmaf(w, s.y, k * v.y), fmaf(w, s.z, k * v.z), fmaf(w, s.w, k * v.w)};
          const float4 rd = has_bonus ? s : n;
          acc.x = fmaf(q, rd.x, acc.x); acc.y = fmaf(q, rd.y, acc.y);
          acc.z = fmaf(q, rd.z, acc.z); acc.w = fmaf(q, rd.w, acc.w);
          if (live) *reinterpret_cast<float4*>(at) = n;
        }
        *reinterpret_cast<float4*>(so + rg * dv + 4 * cg) = acc;
      } else {
        const float v = sv[cg];
        float acc = 0.f;
        for (int r = rg; r < dk; r += rgs) {
          float* at = st + (int64_t)r * dv + cg;
          const float s = fresh ? 0.f : *at;
          const float n = fmaf(sw[r], s, sk[r] * v);
          acc = fmaf(sq[r], has_bonus ? s : n, acc);
          if (live) *at = n;
        }
        so[rg * dv + cg] = acc;
      }
    }
  }
  __syncthreads();
  const float bonus = s_bonus;
  float ss = 0.f;
  for (int d = threadIdx.x; d < dv; d += 256) {
    float o = has_bonus ? bonus * sv[d] : 0.f;
    for (int r = 0; r < rgs; ++r) o += so[r * dv + d];
    so[d] = o;  // (column d is this thread's alone)
    ss = fmaf(o, o, ss);
  }
  const float r = 1.f / sqrtf(block_sum(ss, red) / dv + p.eps);
  for (int d = threadIdx.x; d < dv; d += 256) {
    const bool first = d == tid;
    const float z = first ? gate0 : T::to_float(((const S*)p.gate)[(int64_t)row * p.gate_stride + head * dv + d]);
    const float w = first ? weight0 : p.norm_weight[head * p.norm_head_stride + d];
    const float silu = z / (1.f + expf(-z));
    ((S*)p.out)[(int64_t)row * p.out_stride + head * dv + d] = T::from_float(so[d] * r * w * silu * p.out_scale);
  }
}

// 64-channel groups of the state and 16-column tiles of a value slice
static int key_groups(int dk) { return dk <= 64 ? 1 : dk <= 128 ? 2 : 4; }
static int value_tiles(int dk, int dv) {
  const int most = dk <= 128 ? 8 : 4;
  int n = 1;
  while (n < most && n * 16 < dv) n *= 2;
  return n;
}
static int value_slices(int dk, int dv) { return (dv + 16 * value_tiles(dk, dv) - 1) / (16 * value_tiles(dk, dv)); }

constexpr int mix_wgs_per_cu(int NT, int NV) { return NT == 1 && NV <= 4 ? 3 : 2; }  // (registers; the LDS holds as many)

// Chunks per segment: sequences are cut when (sequence, head, value slice) triples alone leave CUs idle, into as many
// segments as run at once
static int segment_chunks(int rows, int heads, int dk, int dv, int max_query_len) {
  const int chunks = (max_query_len + kChunk - 1) / kChunk;
  const int64_t long_seqs = (rows + max_query_len - 1) / max_query_len;
  const int64_t wide = long_seqs * heads * value_slices(dk, dv);
  const int64_t segs = 256 * mix_wgs_per_cu(key_groups(dk), value_tiles(dk, dv)) / wide;
  const int per = segs < 2 ? chunks : (int)((chunks + segs - 1) / segs);
  return per < 8 ? 8 : per;
}
static int64_t segment_slots(int rows, int num_seqs, int per, int max_query_len) {
  return max_query_len <= per * kChunk ? 0 : (int64_t)rows / (kChunk * per) + num_seqs + 1;
}

template <typename T, int NT, int NV>
static void launch_mix(const MixParams& p, hipStream_t s) {
  constexpr int smem = mix_smem_floats(NT, NV) * 4;
  const dim3 grid(p.heads, value_slices(p.dk, p.dv), p.num_seqs * p.max_segs);
  if (p.max_segs > 1) {
    hipLaunchKernelGGL((chunk_mix_kernel<T, NT, NV, true>), grid, dim3(256), 0, s, p);
    hipLaunchKernelGGL(chunk_combine_kernel, dim3((unsigned)(((int64_t)p.dk * p.dv + 255) / 256), p.heads, p.num_seqs),
                       dim3(256), 0, s, p, 64 * NT);
  }
  if (smem > 64 * 1024)
    (void)hipFuncSetAttribute((const void*)chunk_mix_kernel<T, NT, NV, false>, hipFuncAttributeMaxDynamicSharedMemorySize, smem);
  hipLaunchKernelGGL((chunk_mix_kernel<T, NT, NV, false>), grid, dim3(256), smem, s, p);
}

template <typename T>
static void launch_mix_sized(const MixParams& p, hipStream_t s) {
  const int nv = value_tiles(p.dk, p.dv);
  switch (key_groups(p.dk) * 16 + nv) {
    case 17: launch_mix<T, 1, 1>(p, s); break;
    case 18: launch_mix<T, 1, 2>(p, s); break;
    case 20: launch_mix<T, 1, 4>(p, s); break;
    case 24: launch_mix<T, 1, 8>(p, s); break;
    case 33: launch_mix<T, 2, 1>(p, s); break;
    case 34: launch_mix<T, 2, 2>(p, s); break;
    case 36: launch_mix<T, 2, 4>(p, s); break;
    case 40: launch_mix<T, 2, 8>(p, s); break;
    case 65: launch_mix<T, 4, 1>(p, s); break;
    case 66: launch_mix<T, 4, 2>(p, s); break;
    default: launch_mix<T, 4, 4>(p, s); break;
  }
}

}  // namespace lvllm

using namespace lvllm;

extern "C" int lvllm_log_decay(float* out, const void* u, int64_t u_stride, const float* a_t, const float* bias, int kind,
                               float inv_tau, int rows, int rank, int channels, int dtype, void* stream) {
  if (rows == 0) return 0;
  LV_CHECK(kind == kDecayLogSigmoid || kind == kDecayNegExp, "unknown decay kind");
  LV_CHECK(rank > 0 && rank <= 512 && channels > 0, "rank must be in 1 .. 512");
  const size_t smem = (size_t)kDecayRows * (((rank + 3) & ~3) + 1) * 4;
  const int ny = (rows + kDecayRows - 1) / kDecayRows;
  LV_CHECK(ny <= 65535, "too many rows");
  LV_DISPATCH_DTYPE(dtype, {
    using S = scalar_t::store_t;
    if (smem > 64 * 1024)
      (void)hipFuncSetAttribute((const void*)log_decay_kernel<scalar_t>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)smem);
    hipLaunchKernelGGL((log_decay_kernel<scalar_t>), dim3((channels + kDecayCols - 1) / kDecayCols, ny), dim3(256), smem,
                       (hipStream_t)stream, out, (const S*)u, u_stride, a_t, bias, kind,
                       inv_tau, rows, rank, channels);
  });
  LV_LAUNCH_CHECK();
  return 0;
}

extern "C" int lvllm_recurrent_scan(float* o, const void* q, const void* k, const void* v, int64_t q_stride,
                                    int64_t k_stride, int64_t v_stride, const float* log_decay, const float* bonus,
                                    float q_scale, float* state, int64_t state_stride, const int32_t* state_slots,
                                    int num_slots, const int32_t* query_start_loc, const int32_t* seq_lens, int num_seqs,
                                    int heads, int dk, int dv, int dtype, void* stream) {
  if (num_seqs == 0) return 0;
  LV_CHECK(dk > 0 && dk <= 256 && dv > 0, "key size must be in 1 .. 256");
  LV_CHECK(state_stride >= (int64_t)heads * dk * dv, "state slots overlap");
  const ScanParams p{o, q, k, v, q_stride, k_stride, v_stride, log_decay, bonus, q_scale, state, state_stride,
                     state_slots, query_start_loc, seq_lens, num_slots, heads, dk, dv};
  hipStream_t s = (hipStream_t)stream;
  LV_DISPATCH_DTYPE(dtype, {
    if (dk <= 32) launch_scan<scalar_t, 8>(p, num_seqs, s);
    else if (dk <= 64) launch_scan<scalar_t, 16>(p, num_seqs, s);
    else if (dk <= 128) launch_scan<scalar_t, 32>(p, num_seqs, s);
    else launch_scan<scalar_t, 64>(p, num_seqs, s);
  });
  LV_LAUNCH_CHECK();
  return 0;
}

extern "C" int64_t lvllm_recurrent_mix_workspace_bytes(int rows, int num_seqs, int heads, int dk, int dv, int max_query_len) {
  if (max_query_len <= 1) return 0;
  const int per = segment_chunks(rows, heads, dk, dv, max_query_len);
  const int64_t segs = segment_slots(rows, num_seqs, per, max_query_len) * heads;
  const int64_t o = value_slices(dk, dv) > 1 ? (int64_t)rows * heads * dv : 0;
  return ((int64_t)rows * heads * dk + segs * ((int64_t)dk * dv + 64 * key_groups(dk)) + o) * 4;
}

extern "C" int lvllm_recurrent_mix(void* out, int64_t out_stride, const void* q, const void* k, const void* v,
                                   int64_t q_stride, int64_t k_stride, int64_t v_stride, const void* u, int64_t u_stride,
                                   const float* a_t, const float* decay_bias, int rank, int kind, float inv_tau,
                                   const float* bonus, float q_scale, const void* gate, int64_t gate_stride,
                                   const float* norm_weight, int norm_head_stride, float eps, float out_scale, float* state,
                                   int64_t state_stride, const int32_t* state_slots, int num_slots,
                                   const int32_t* query_start_loc, const int32_t* seq_lens, int num_seqs, int rows,
                                   int heads, int dk, int dv, int max_query_len, void* workspace,
                                   int64_t workspace_bytes, int dtype, void* stream) {
  if (num_seqs == 0 || rows == 0) return 0;
  LV_CHECK(dk > 0 && dk <= 256 && dv > 0 && dv <= 1024, "key size must be in 1 .. 256, value size in 1 .. 1024");
  LV_CHECK(kind == kDecayLogSigmoid || kind == kDecayNegExp, "unknown decay kind");
  LV_CHECK(rank > 0 && rank <= 512, "rank must be in 1 .. 512");
  LV_CHECK(state_stride >= (int64_t)heads * dk * dv && ((dv & 3) != 0 || (state_stride & 3) == 0),
           "state slots overlap or are unaligned");
  LV_CHECK(num_seqs <= 65535 && heads <= 65535, "too many sequences or heads");
  MixParams p{};
  p.q = q; p.k = k; p.v = v; p.q_stride = q_stride; p.k_stride = k_stride; p.v_stride = v_stride;
  p.u = u; p.u_stride = u_stride; p.a_t = a_t; p.decay_bias = decay_bias; p.kind = kind; p.rank = rank; p.inv_tau = inv_tau;
  p.bonus = bonus; p.q_scale = q_scale; p.state = state; p.state_stride = state_stride; p.state_slots = state_slots;
  p.query_start_loc = query_start_loc; p.seq_lens = seq_lens; p.num_seqs = num_seqs; p.num_slots = num_slots;
  p.heads = heads; p.dk = dk; p.dv = dv; p.out = out; p.out_stride = out_stride; p.gate = gate; p.gate_stride = gate_stride;
  p.norm_weight = norm_weight; p.norm_head_stride = norm_head_stride; p.eps = eps; p.out_scale = out_scale;
  hipStream_t s = (hipStream_t)stream;
  if (max_query_len <= 1) {  // every sequence brings one token: sequence s owns row s
    const int cgs = (dv & 3) == 0 ? dv / 4 : dv, per = cgs < 256 ? cgs : 256, rgs = 256 / per;
    const int groups = rgs * dv > 256 ? rgs * dv : 256;
    const size_t smem = (size_t)(3 * dk + rank + 3 + dv + groups + 8) * sizeof(float);  // (at most 16 KB)
    const int pre = (dv & 3) == 0 ? (dk + rgs - 1) / rgs : 1 << 20;  // state rows per thread
    const dim3 grid(heads, num_seqs);
    LV_DISPATCH_DTYPE(dtype, {
      if (pre <= 4) hipLaunchKernelGGL((recurrent_decode_kernel<scalar_t, 4>), grid, dim3(256), smem, s, p);
      else if (pre <= 8) hipLaunchKernelGGL((recurrent_decode_kernel<scalar_t, 8>), grid, dim3(256), smem, s, p);
      else if (pre <= 16) hipLaunchKernelGGL((recurrent_decode_kernel<scalar_t, 16>), grid, dim3(256), smem, s, p);
      else hipLaunchKernelGGL((recurrent_decode_kernel<scalar_t, 0>), grid, dim3(256), smem, s, p);
    });
    LV_LAUNCH_CHECK();
    return 0;
  }
  LV_CHECK(dtype == LVLLM_BF16 || dtype == LVLLM_F32, "bfloat16 or float32");
  LV_CHECK(workspace != nullptr &&
               workspace_bytes >= lvllm_recurrent_mix_workspace_bytes(rows, num_seqs, heads, dk, dv, max_query_len),
           "workspace too small (see lvllm_recurrent_mix_workspace_bytes)");
  float* ws = (float*)workspace;
  p.log_decay = ws;
  ws += (int64_t)rows * heads * dk;
  p.seg_chunks = segment_chunks(rows, heads, dk, dv, max_query_len);
  p.max_segs = (max_query_len + kChunk * p.seg_chunks - 1) / (kChunk * p.seg_chunks);
  LV_CHECK((int64_t)num_seqs * p.max_segs <= 65535, "too many sequences or too long portions");
  const int64_t segs = segment_slots(rows, num_seqs, p.seg_chunks, max_query_len) * heads;
  p.seg_decay = ws;
  ws += segs * 64 * key_groups(dk);
  p.seg_state = ws;
  ws += segs * dk * dv;
  if (value_slices(dk, dv) > 1) p.o = ws;
  const int esize = dtype == LVLLM_F32 ? 4 : 2;
  p.vec_in = ((dv | v_stride | gate_stride) & 3) == 0 && (((uintptr_t)v | (uintptr_t)gate) & (4 * esize - 1)) == 0;
  p.vec_out = ((dv | out_stride) & 3) == 0 && ((uintptr_t)out & (4 * esize - 1)) == 0;
  if (int rc = lvllm_log_decay((float*)workspace, u, u_stride, a_t, decay_bias, kind, inv_tau, rows, rank, heads * dk, dtype, stream))
    return rc;
  if (dtype == LVLLM_BF16) launch_mix_sized<BF16>(p, s);
  else launch_mix_sized<F32>(p, s);
  LV_LAUNCH_CHECK();
  if (p.o == nullptr) return 0;
  return lvllm_head_norm_gate(out, out_stride, p.o, gate, gate_stride, norm_weight, norm_head_stride, eps, out_scale, rows,
                              heads, dv, dtype, stream);
}
