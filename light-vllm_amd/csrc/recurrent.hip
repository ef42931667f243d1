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
//   * everything else: chunks of 16 tokens on fp32 MFMAs; long sequences that alone would not fill the chip are cut into
//     segments of chunks, whose states are found first.  A parallel pass (chunk_prepare_kernel) computes per (chunk, head)
//     the decays and all that does not depend on the state: q scaled by the decay from the chunk's start, k scaled by the
//     decay to its end, the masked 16 x 16 products inside the chunk.  A sequential pass (chunk_scan_kernel) then needs
//     17 MFMAs per chunk and wave: its state tiles are MFMA accumulators AND, without a move, the B operands of the
//     read-out (k-step r of a tile contracts rows {r, 4 + r, 8 + r, 12 + r}: accumulator register r of every lane).
//   Inside a chunk the decay between two tokens is the product of two factors measured from the chunk's middle; a
//   workgroup whose channels decay too fast for that (a factor would leave fp32's range) takes the products pair by pair.
//
// Everything but the projections' results (q, k, v, the low-rank input) is fp32: decays and their logarithms, the state,
// the read-out.  Rows are the new tokens of `num_seqs` sequences back to back (query_start_loc); a sequence whose tokens
// are all in this step (seq_lens == its rows) starts from a zero state, every other one from its slot.
#include "common.h"

namespace lvllm {

enum { kDecayLogSigmoid = 0, kDecayNegExp = 1 };

__device__ __forceinline__ float log_decay_of(float z, int kind, float inv_tau) {
  if (kind == kDecayNegExp) return -expf(fminf(z, 9.f));  // (exp(-exp(9)) is 0: a finite logarithm keeps sums finite)
  return (fminf(z, 0.f) - log1pf(expf(-fabsf(z)))) * inv_tau;
}

// e^x for x <= 0 (and for the bounded positive factors of a chunk): 2^(x log2 e) with the product's rounding error put back
__device__ __forceinline__ float exp_of(float x) {
  const float t = x * 1.44269502e+0f;
  const float lo = fmaf(x, 1.44269502e+0f, -t) + x * 1.92596299e-8f;
  const float r = __builtin_amdgcn_exp2f(t);
  return fmaf(r, lo * 0.693147182f, r);
}

// ---- ln w [rows, channels] ---------------------------------------------------------------------------------------
constexpr int kDecayRows = 8;
template <typename T>
__global__ __launch_bounds__(256) void log_decay_kernel(float* __restrict__ out, const typename T::store_t* __restrict__ u,
                                                        const int64_t u_stride, const float* __restrict__ a_t,  // [rank, channels]
                                                        const float* __restrict__ bias, const int kind,
                                                        const float inv_tau, const int rows, const int rank,
                                                        const int channels) {
  extern __shared__ float su[];  // [kDecayRows][rank]
  const int row0 = blockIdx.y * kDecayRows;
  const int nr = min(kDecayRows, rows - row0);
  for (int i = threadIdx.x; i < kDecayRows * rank; i += blockDim.x) {
    const int r = i / rank, c = i - r * rank;
    float f = r < nr ? T::to_float(u[(row0 + r) * u_stride + c]) : 0.f;
    su[i] = kind == kDecayNegExp ? tanhf(f) : f;
  }
  __syncthreads();
  const int ch = blockIdx.x * blockDim.x + threadIdx.x;
  if (ch >= channels) return;
  float acc[kDecayRows];
#pragma unroll
  for (int r = 0; r < kDecayRows; ++r) acc[r] = 0.f;
  for (int c = 0; c < rank; ++c) {
    const float w = a_t[(int64_t)c * channels + ch];
#pragma unroll
    for (int r = 0; r < kDecayRows; ++r) acc[r] = fmaf(su[r * rank + c], w, acc[r]);
  }
  const float b = bias[ch];
#pragma unroll
  for (int r = 0; r < kDecayRows; ++r)
    if (r < nr) out[(int64_t)(row0 + r) * channels + ch] = log_decay_of(acc[r] + b, kind, inv_tau);
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
typedef float r_f32x4_t __attribute__((ext_vector_type(4)));
__device__ __forceinline__ r_f32x4_t mfma_f32(float a, float b, r_f32x4_t c) {
  return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0);
}
constexpr int kChunk = 16;
constexpr float kMaxHalfDecay = 60.f;  // ln of the largest factor measured from the middle of a chunk

// per (chunk, head): floats of the workspace
__host__ __device__ constexpr int chunk_floats(int dkp) { return 2 * kChunk * dkp + kChunk * kChunk + dkp; }

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
  // chunked body
  float* ws;              // [chunk slots, heads, chunk_floats(dkp)]
  float* o;               // [rows, heads, dv]
  int seg_chunks, max_segs;  // chunks per segment, segments of the longest sequence (1: not cut)
  float* seg_state;       // [segment slots, heads, dk, dv]
  float* seg_decay;       // [segment slots, heads, dkp]
};

// Chunk ci of sequence s has slot query_start_loc[s] / 16 + s + ci: unique, and monotonic in s.
__device__ __forceinline__ int chunk_slot_base(const int32_t* qsl, int s) { return qsl[s] / kChunk + s; }
__device__ __forceinline__ int seg_slot_base(const MixParams& p, int s) {
  return p.query_start_loc[s] / (kChunk * p.seg_chunks) + s;
}

// One workgroup (4 waves) per (chunk slot, head); wave w owns key channels [w * 16 * NT, (w + 1) * 16 * NT).
template <typename T, int NT>
__global__ __launch_bounds__(256) void chunk_prepare_kernel(const MixParams p) {
  using S = typename T::store_t;
  constexpr int DKP = 64 * NT;
  constexpr int LD = DKP + 4;  // row stride of the LDS images (bank spread of the 16-byte reads)
  extern __shared__ float sm[];
  float* sq = sm;                  // [16][LD]; before that the low-rank input f(u) [16][rank_ld]
  float* sk = sq + kChunk * LD;    // [16][LD]
  float* sb = sk + kChunk * LD;    // [16][LD]: ln w (slow path)
  float* spart = sb + kChunk * LD; // [4][16][16]
  float* sdiag = spart + 4 * 256;  // [4][16]
  const int head = blockIdx.y;
  int lo = 0, hi = p.num_seqs;  // the sequence that owns this chunk slot: the last s with base(s) <= slot
  while (lo < hi) {
    const int mid = (lo + hi) >> 1;
    if (chunk_slot_base(p.query_start_loc, mid) <= (int)blockIdx.x) lo = mid + 1;
    else hi = mid;
  }
  const int seq = lo - 1;
  if (seq < 0) return;
  const int qbeg = p.query_start_loc[seq], qlen = p.query_start_loc[seq + 1] - qbeg;
  const int t0 = ((int)blockIdx.x - chunk_slot_base(p.query_start_loc, seq)) * kChunk;
  if (t0 >= qlen) return;
  const int nt = min(kChunk, qlen - t0);
  const int64_t row0 = qbeg + t0;
  const int lane = threadIdx.x & 63;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int g = lane >> 4, c = lane & 15;
  float* ws = p.ws + ((int64_t)blockIdx.x * p.heads + head) * chunk_floats(DKP);
  float* w_q = ws;                       // [16 tokens][DKP]
  float* w_k = w_q + kChunk * DKP;       // [DKP][16 tokens]
  float* w_a = w_k + kChunk * DKP;       // [16][16]
  float* w_end = w_a + kChunk * kChunk;  // [DKP]

  // q and k of this lane (tokens 4g .. 4g + 3 of each channel tile), in flight while the decays are computed; addresses are
  // clamped instead of predicated and the values masked when they are used
  S qraw[NT][4], kraw[NT][4];
#pragma unroll
  for (int i = 0; i < NT; ++i) {
    const int chc = min((wave * NT + i) * 16 + c, p.dk - 1);
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int64_t row = row0 + min(4 * g + r, nt - 1);
      qraw[i][r] = ((const S*)p.q)[row * p.q_stride + head * p.dk + chc];
      kraw[i][r] = ((const S*)p.k)[row * p.k_stride + head * p.dk + chc];
    }
  }
  // z[token, channel] = f(u) . a_t on MFMAs: A operand lane (token = c, k = g), B operand lane (k = g, channel = c)
  const int rank4 = (p.rank + 3) & ~3, rank_ld = rank4 + 1;
  for (int i = threadIdx.x; i < kChunk * rank4; i += 256) {
    const int t = i / rank4, kk = i - t * rank4;
    float f = 0.f;
    if (t < nt && kk < p.rank) f = T::to_float(((const S*)p.u)[(row0 + t) * p.u_stride + kk]);
    sq[t * rank_ld + kk] = p.kind == kDecayNegExp ? tanhf(f) : f;
  }
  __syncthreads();
  r_f32x4_t z[NT];
#pragma unroll
  for (int i = 0; i < NT; ++i) z[i] = r_f32x4_t{0.f, 0.f, 0.f, 0.f};
  const int64_t a_step = (int64_t)p.heads * p.dk;
  const float* a_ch[NT];
#pragma unroll
  for (int i = 0; i < NT; ++i) a_ch[i] = p.a_t + head * p.dk + min((wave * NT + i) * 16 + c, p.dk - 1);
#pragma unroll 4
  for (int k0 = 0; k0 < rank4; k0 += 4) {
    const float a = sq[c * rank_ld + k0 + g];
    const int64_t at = min(k0 + g, p.rank - 1) * a_step;  // (beyond the rank: f(u) is zero)
#pragma unroll
    for (int i = 0; i < NT; ++i) z[i] = mfma_f32(a, a_ch[i][at], z[i]);
  }
  // lane (channel c of its tile, tokens 4g .. 4g + 3): ln w, then its sums over ranges of the chunk's tokens.  Every range
  // is summed by itself: a difference of two running sums would lose the small decays behind a large one.
  float lw[NT][4], read[NT][4], left[NT][4], h1[NT], h2[NT];  // h1, h2: the two halves; read: chunk's start -> what token t reads; left: token t -> end
  float half_q[NT][4], half_k[NT][4];                  // the middle of the chunk -> what token t reads; token t -> the middle
  const bool has_bonus = p.bonus != nullptr;
  bool fast = true;
#pragma unroll
  for (int i = 0; i < NT; ++i) {
    const int ch = (wave * NT + i) * 16 + c;
    const float bias = ch < p.dk ? p.decay_bias[head * p.dk + ch] : 0.f;
    float(&l)[4] = lw[i];
#pragma unroll
    for (int r = 0; r < 4; ++r)
      l[r] = (4 * g + r < nt && ch < p.dk) ? log_decay_of(z[i][r] + bias, p.kind, p.inv_tau) : 0.f;
    const float upto[4] = {l[0], l[0] + l[1], (l[0] + l[1]) + l[2], (l[0] + l[1]) + (l[2] + l[3])};
    const float after[4] = {l[1] + (l[2] + l[3]), l[2] + l[3], l[3], 0.f};
    const float g0 = __shfl(upto[3], c), g1 = __shfl(upto[3], 16 + c), g2 = __shfl(upto[3], 32 + c), g3 = __shfl(upto[3], 48 + c);
    const float before_g = g == 0 ? 0.f : g == 1 ? g0 : g == 2 ? g0 + g1 : g0 + g1 + g2;
    const float after_g = g == 3 ? 0.f : g == 2 ? g3 : g == 1 ? g2 + g3 : g1 + (g2 + g3);
    const float in_half = g == 0 ? g1 : g == 3 ? g2 : 0.f;  // the group of this half between this one and the middle
    h1[i] = g0 + g1;
    h2[i] = g2 + g3;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const float upto_read = has_bonus ? (r == 0 ? 0.f : upto[r == 0 ? 0 : r - 1]) : upto[r];
      const float from_read = has_bonus ? after[r] + l[r] : after[r];
      read[i][r] = before_g + upto_read;
      left[i][r] = after[r] + after_g;
      half_q[i][r] = g < 2 ? -(from_read + in_half) : in_half + upto_read;
      half_k[i][r] = g < 2 ? after[r] + in_half : -(in_half + upto[r]);
    }
    fast = fast && -h1[i] < kMaxHalfDecay && -h2[i] < kMaxHalfDecay;
  }
  const bool slow = __syncthreads_or(!fast);  // (the low-rank input in LDS has been read)
  float diag[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int i = 0; i < NT; ++i) {
    const int ch = (wave * NT + i) * 16 + c;
    const bool ok = ch < p.dk;
    const float bon = (has_bonus && ok) ? p.bonus[head * p.dk + ch] : 0.f;
    const float to_mid = exp_of(h1[i]), from_mid = exp_of(h2[i]);
    float kd[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int t = 4 * g + r;
      const bool live = ok && t < nt;
      const float qv = live ? T::to_float(qraw[i][r]) * p.q_scale : 0.f;
      const float kv = live ? T::to_float(kraw[i][r]) : 0.f;
      if (slow) {
        w_q[t * DKP + ch] = qv * exp_of(read[i][r]);
        kd[r] = kv * exp_of(left[i][r]);
        sq[t * LD + ch] = qv;
        sk[t * LD + ch] = kv;
        sb[t * LD + ch] = lw[i][r];
      } else {
        const float qh = qv * exp_of(half_q[i][r]), kh = kv * exp_of(half_k[i][r]);
        w_q[t * DKP + ch] = qh * to_mid;
        kd[r] = kh * from_mid;
        sq[t * LD + ch] = qh;
        sk[t * LD + ch] = kh;
      }
      diag[r] = fmaf(qv * bon, kv, diag[r]);
    }
    *reinterpret_cast<float4*>(w_k + ch * kChunk + 4 * g) = float4{kd[0], kd[1], kd[2], kd[3]};
    if (g == 0) w_end[ch] = exp_of(h1[i] + h2[i]);
  }
  if (has_bonus) {
#pragma unroll
    for (int r = 0; r < 4; ++r) {
#pragma unroll
      for (int m = 1; m < 16; m <<= 1) diag[r] += __shfl_xor(diag[r], m);
      if (c == 0) sdiag[wave * 16 + 4 * g + r] = diag[r];
    }
  }
  if (!slow) {
    // this wave's channels only: what it wrote itself, no barrier needed for other waves' parts
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
  }
  __syncthreads();
  const int ti = threadIdx.x >> 4, tj = threadIdx.x & 15;
  const bool below = has_bonus ? tj < ti : tj <= ti;
  float a = 0.f;
  if (below) {
    if (slow) {
      for (int ch = 0; ch < p.dk; ++ch) {
        float between = 0.f;
        for (int t = tj + 1; t < (has_bonus ? ti : ti + 1); ++t) between += sb[t * LD + ch];
        a = fmaf(sq[ti * LD + ch] * exp_of(between), sk[tj * LD + ch], a);
      }
    } else {
      a = (spart[threadIdx.x] + spart[256 + threadIdx.x]) + (spart[512 + threadIdx.x] + spart[768 + threadIdx.x]);
    }
  } else if (has_bonus && ti == tj) {
    a = (sdiag[ti] + sdiag[16 + ti]) + (sdiag[32 + ti] + sdiag[48 + ti]);
  }
  w_a[threadIdx.x] = a;
}

// One workgroup per (sequence, head, 16 * NV value columns), walking chunks in order.  Wave w holds state rows
// [w * 16 * NT, (w + 1) * 16 * NT) as accumulator tiles; the four waves' partial read-outs meet in LDS.
// Sequences too few to fill the chip are cut into segments of seg_chunks chunks:
//   kScanWhole     no segments: the state comes from the slot and goes back there;
//   kScanStates    each segment but the last, from a zero state: its last state and the product of its decays;
//   (chunk_combine_kernel turns those into every segment's first state)
//   kScanSegments  each segment from its first state; the last one stores the slot.
enum { kScanWhole, kScanStates, kScanSegments };
template <typename T, int NT, int NV, int MODE>
__global__ __launch_bounds__(256) void chunk_scan_kernel(const MixParams p) {
  using S = typename T::store_t;
  constexpr int DKP = 64 * NT;
  __shared__ float so[MODE == kScanStates ? 1 : 2][4][kChunk][16 * NV];
  const int head = blockIdx.x, v0 = blockIdx.y * 16 * NV;
  const int seq = MODE == kScanWhole ? blockIdx.z : blockIdx.z / p.max_segs;
  const int seg = MODE == kScanWhole ? 0 : blockIdx.z - seq * p.max_segs;
  const int qbeg = p.query_start_loc[seq], qlen = p.query_start_loc[seq + 1] - qbeg;
  if (qlen <= 0) return;
  const int all_chunks = (qlen + kChunk - 1) / kChunk;
  const int first = MODE == kScanWhole ? 0 : seg * p.seg_chunks;
  const int last = MODE == kScanWhole ? all_chunks : min(first + p.seg_chunks, all_chunks);
  if (first >= all_chunks || (MODE == kScanStates && last == all_chunks)) return;
  const int lane = threadIdx.x & 63;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int g = lane >> 4, c = lane & 15;
  const int slot = p.state_slots[seq];
  const bool live = slot >= 0 && slot < p.num_slots;
  float* st = p.state + (int64_t)(live ? slot : 0) * p.state_stride + (int64_t)head * p.dk * p.dv;
  const bool fresh = p.seq_lens[seq] <= qlen || !live;
  const int64_t seg_slot = MODE == kScanWhole ? 0 : seg_slot_base(p, seq) + seg;
  float* seg_st = MODE == kScanWhole ? nullptr : p.seg_state + (seg_slot * p.heads + head) * p.dk * p.dv;
  r_f32x4_t s[NT][NV];
#pragma unroll
  for (int i = 0; i < NT; ++i)
#pragma unroll
    for (int j = 0; j < NV; ++j)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int row = (wave * NT + i) * 16 + 4 * g + r, col = v0 + 16 * j + c;
        const bool in = row < p.dk && col < p.dv;
        if (MODE == kScanWhole) s[i][j][r] = (!fresh && in) ? st[(int64_t)row * p.dv + col] : 0.f;
        else if (MODE == kScanSegments) s[i][j][r] = in ? seg_st[(int64_t)row * p.dv + col] : 0.f;
        else s[i][j][r] = 0.f;
      }
  float4 decays[NT];  // (kScanStates) products of this lane's rows' decays
#pragma unroll
  for (int i = 0; i < NT; ++i) decays[i] = float4{1.f, 1.f, 1.f, 1.f};
  const float* ws0 = p.ws + ((int64_t)chunk_slot_base(p.query_start_loc, seq) * p.heads + head) * chunk_floats(DKP);
  const int64_t ws_step = (int64_t)p.heads * chunk_floats(DKP);

  struct Frag {
    float4 q[NT], k[NT], e[NT];
    float a;
    float v[NV][4];
  };
  auto load = [&](int ci, Frag& f) __attribute__((always_inline)) {
    const float* ws = ws0 + ci * ws_step;
#pragma unroll
    for (int i = 0; i < NT; ++i) {
      const int ch0 = (wave * NT + i) * 16;
      if (MODE != kScanStates) f.q[i] = *reinterpret_cast<const float4*>(ws + c * DKP + ch0 + 4 * g);
      f.k[i] = *reinterpret_cast<const float4*>(ws + kChunk * DKP + (ch0 + c) * kChunk + 4 * g);
      f.e[i] = *reinterpret_cast<const float4*>(ws + 2 * kChunk * DKP + kChunk * kChunk + ch0 + 4 * g);
    }
    if (MODE != kScanStates) f.a = ws[2 * kChunk * DKP + c * kChunk + 4 * g + wave];
#pragma unroll
    for (int j = 0; j < NV; ++j)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int t = ci * kChunk + 4 * g + r, col = v0 + 16 * j + c;
        f.v[j][r] = (t < qlen && col < p.dv)
                        ? T::to_float(((const S*)p.v)[(int64_t)(qbeg + t) * p.v_stride + head * p.dv + col]) : 0.f;
      }
  };
  auto step = [&](int ci, const Frag& f) __attribute__((always_inline)) {
    float(*buf)[kChunk][16 * NV] = so[MODE == kScanStates ? 0 : ci & 1];
#pragma unroll
    for (int j = 0; j < NV; ++j) {
      if (MODE != kScanStates) {
        r_f32x4_t o{0.f, 0.f, 0.f, 0.f};
        // inside the chunk: this wave contracts tokens {4g + wave}
        const float vw = wave == 0 ? f.v[j][0] : wave == 1 ? f.v[j][1] : wave == 2 ? f.v[j][2] : f.v[j][3];
        o = mfma_f32(f.a, vw, o);
#pragma unroll
        for (int i = 0; i < NT; ++i) {
          o = mfma_f32(f.q[i].x, s[i][j][0], o);
          o = mfma_f32(f.q[i].y, s[i][j][1], o);
          o = mfma_f32(f.q[i].z, s[i][j][2], o);
          o = mfma_f32(f.q[i].w, s[i][j][3], o);
        }
#pragma unroll
        for (int r = 0; r < 4; ++r) buf[wave][4 * g + r][16 * j + c] = o[r];
      }
#pragma unroll
      for (int i = 0; i < NT; ++i) {
        r_f32x4_t n = s[i][j];
        n[0] *= f.e[i].x; n[1] *= f.e[i].y; n[2] *= f.e[i].z; n[3] *= f.e[i].w;
        n = mfma_f32(f.k[i].x, f.v[j][0], n);
        n = mfma_f32(f.k[i].y, f.v[j][1], n);
        n = mfma_f32(f.k[i].z, f.v[j][2], n);
        n = mfma_f32(f.k[i].w, f.v[j][3], n);
        s[i][j] = n;
      }
    }
    if (MODE == kScanStates) {
#pragma unroll
      for (int i = 0; i < NT; ++i) {
        decays[i].x *= f.e[i].x; decays[i].y *= f.e[i].y; decays[i].z *= f.e[i].z; decays[i].w *= f.e[i].w;
      }
      return;
    }
    __syncthreads();  // (the buffer of chunk ci + 1 is the other one: it was read before this barrier)
    for (int i = threadIdx.x; i < kChunk * 16 * NV; i += 256) {
      const int t = i / (16 * NV), d = i - t * 16 * NV;
      if (ci * kChunk + t < qlen && v0 + d < p.dv)
        p.o[((int64_t)(qbeg + ci * kChunk + t) * p.heads + head) * p.dv + v0 + d] =
            (buf[0][t][d] + buf[1][t][d]) + (buf[2][t][d] + buf[3][t][d]);
    }
  };
  Frag fa, fb;
  load(first, fa);
  for (int ci = first; ci < last; ci += 2) {
    if (ci + 1 < last) load(ci + 1, fb);
    step(ci, fa);
    if (ci + 1 >= last) break;
    if (ci + 2 < last) load(ci + 2, fa);
    step(ci + 1, fb);
  }
  if (MODE == kScanStates && blockIdx.y == 0 && c == 0) {
#pragma unroll
    for (int i = 0; i < NT; ++i)
      *reinterpret_cast<float4*>(p.seg_decay + (seg_slot * p.heads + head) * DKP + (wave * NT + i) * 16 + 4 * g) = decays[i];
  }
  if (MODE == kScanStates || (live && last == all_chunks)) {
    float* to = MODE == kScanStates ? seg_st : st;
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
// One workgroup per (head, sequence), sequence s owning row s.  Thread (rg, cg): state columns 4 cg .. 4 cg + 3 of rows
// rg, rg + RG, ...  With PRE > 0 the thread's PRE state rows are loaded before anything else, so that the whole state is in
// flight while the decays are computed; PRE = 0 takes any size.
template <typename T, int PRE>
__global__ __launch_bounds__(256) void recurrent_decode_kernel(const MixParams p) {
  using S = typename T::store_t;
  extern __shared__ float sm[];
  const int head = blockIdx.x, seq = blockIdx.y;
  const int row = p.query_start_loc[seq];
  if (p.query_start_loc[seq + 1] - row != 1) return;
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
  float4 pre[PRE > 0 ? PRE : 1];
  if constexpr (PRE > 0) {
#pragma unroll
    for (int i = 0; i < PRE; ++i) {
      pre[i] = float4{0.f, 0.f, 0.f, 0.f};
      const int r = rg + i * rgs;
      if (!fresh && rg < rgs && r < dk) pre[i] = *reinterpret_cast<const float4*>(st + (int64_t)r * dv + 4 * cg0);
    }
  }
  float* sq = sm;            // [dk]
  float* sk = sq + dk;       // [dk]
  float* sw = sk + dk;       // [dk]
  float* su = sw + dk;       // [rank]
  float* sv = sm + ((3 * dk + p.rank + 3) & ~3);  // [dv], 16-byte aligned
  float* so = sv + dv;       // [row groups][dv]; before that the parts of z [max(1, 256 / dk)][dk]
  __shared__ float red[16];
  __shared__ float s_bonus;
  for (int i = threadIdx.x; i < p.rank; i += 256) {
    const float f = T::to_float(((const S*)p.u)[(int64_t)row * p.u_stride + i]);
    su[i] = p.kind == kDecayNegExp ? tanhf(f) : f;
  }
  for (int i = threadIdx.x; i < dv; i += 256) sv[i] = T::to_float(((const S*)p.v)[(int64_t)row * p.v_stride + head * dv + i]);
  for (int i = threadIdx.x; i < dk; i += 256) {
    sq[i] = T::to_float(((const S*)p.q)[(int64_t)row * p.q_stride + head * dk + i]) * p.q_scale;
    sk[i] = T::to_float(((const S*)p.k)[(int64_t)row * p.k_stride + head * dk + i]);
  }
  __syncthreads();
  const int parts = dk >= 256 ? 1 : 256 / dk, part_len = (p.rank + parts - 1) / parts;  // z: the rank cut into parts
  {
    const int part = threadIdx.x / dk, ch = threadIdx.x - part * dk;  // (dk <= 256)
    if (part < parts) {
      const int r1 = min((part + 1) * part_len, p.rank);
      const float* a = p.a_t + head * dk + ch;
      const int64_t a_step = (int64_t)p.heads * dk;
      float z = 0.f;
#pragma unroll 8
      for (int r = part * part_len; r < r1; ++r) z = fmaf(su[r], a[r * a_step], z);
      so[part * dk + ch] = z;
    }
  }
  __syncthreads();
  float bsum = 0.f;
  for (int i = threadIdx.x; i < dk; i += 256) {
    float z = p.decay_bias[head * dk + i];
    for (int q = 0; q < parts; ++q) z += so[q * dk + i];
    sw[i] = expf(log_decay_of(z, p.kind, p.inv_tau));
    if (p.bonus != nullptr) bsum = fmaf(sq[i] * p.bonus[head * dk + i], sk[i], bsum);
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
          if (live) *reinterpret_cast<float4*>(st + (int64_t)r * dv + 4 * cg0) = n;
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
    const float z = T::to_float(((const S*)p.gate)[(int64_t)row * p.gate_stride + head * dv + d]);
    const float silu = z / (1.f + expf(-z));
    ((S*)p.out)[(int64_t)row * p.out_stride + head * dv + d] =
        T::from_float(so[d] * r * p.norm_weight[head * p.norm_head_stride + d] * silu * p.out_scale);
  }
}

// Chunks per segment: sequences are cut when (sequence, head, value slice) triples alone leave CUs idle
static int segment_chunks(int rows, int heads, int dv, int max_query_len) {
  const int chunks = (max_query_len + kChunk - 1) / kChunk;
  const int64_t long_seqs = (rows + max_query_len - 1) / max_query_len;
  const int64_t wide = long_seqs * heads * ((dv + 63) / 64);  // workgroups of 64 columns
  int per = chunks;
  while (per > 8 && wide * ((chunks + per - 1) / per) < 1024) per = (per + 1) / 2;
  return per < 8 ? 8 : per;
}

template <typename T, int NT, int NV>
static void launch_scans(const MixParams& p, hipStream_t s) {
  const int ny = ((p.dv + 15) / 16 + NV - 1) / NV;
  if (p.max_segs <= 1) {
    hipLaunchKernelGGL((chunk_scan_kernel<T, NT, NV, kScanWhole>), dim3(p.heads, ny, p.num_seqs), dim3(256), 0, s, p);
    return;
  }
  const dim3 grid(p.heads, ny, p.num_seqs * p.max_segs);
  hipLaunchKernelGGL((chunk_scan_kernel<T, NT, NV, kScanStates>), grid, dim3(256), 0, s, p);
  hipLaunchKernelGGL(chunk_combine_kernel, dim3((unsigned)(((int64_t)p.dk * p.dv + 255) / 256), p.heads, p.num_seqs),
                     dim3(256), 0, s, p, 64 * NT);
  hipLaunchKernelGGL((chunk_scan_kernel<T, NT, NV, kScanSegments>), grid, dim3(256), 0, s, p);
}

template <typename T, int NT>
static void launch_chunks(const MixParams& p, int rows, hipStream_t s) {
  constexpr int LD = 64 * NT + 4;
  const int images = 3 * kChunk * LD + 4 * 256 + 64, low_rank = kChunk * (((p.rank + 3) & ~3) + 1);
  const size_t smem = (size_t)(images > low_rank ? images : low_rank) * sizeof(float);
  if (smem > 64 * 1024)
    (void)hipFuncSetAttribute((const void*)chunk_prepare_kernel<T, NT>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)smem);
  hipLaunchKernelGGL((chunk_prepare_kernel<T, NT>), dim3(rows / kChunk + p.num_seqs + 1, p.heads), dim3(256), smem, s, p);
  const int tiles = (p.dv + 15) / 16;
  // 16 columns per workgroup fill the chip with few (segment, head) pairs; wider slices re-read q, k and the in-chunk
  // products less often
  const int64_t wgs = (int64_t)p.heads * p.num_seqs * p.max_segs * tiles;
  if (wgs <= 512 || tiles == 1) launch_scans<T, NT, 1>(p, s);
  else if (wgs <= 2048 || tiles == 2 || NT > 2) launch_scans<T, NT, 2>(p, s);
  else launch_scans<T, NT, (NT > 2 ? 2 : 4)>(p, s);
}

}  // namespace lvllm

using namespace lvllm;

extern "C" int lvllm_log_decay(float* out, const void* u, int64_t u_stride, const float* a_t, const float* bias, int kind,
                               float inv_tau, int rows, int rank, int channels, int dtype, void* stream) {
  if (rows == 0) return 0;
  LV_CHECK(kind == kDecayLogSigmoid || kind == kDecayNegExp, "unknown decay kind");
  LV_CHECK(rank > 0 && rank <= 1024 && channels > 0, "rank must be in 1 .. 1024");
  const int ny = (rows + kDecayRows - 1) / kDecayRows;
  LV_CHECK(ny <= 65535, "too many rows");
  LV_DISPATCH_DTYPE(dtype, {
    using S = scalar_t::store_t;
    hipLaunchKernelGGL((log_decay_kernel<scalar_t>), dim3((channels + 255) / 256, ny), dim3(256),
                       (size_t)kDecayRows * rank * 4, (hipStream_t)stream, out, (const S*)u, u_stride, a_t, bias, kind,
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

static int padded_dk(int dk) { return (dk + 63) / 64 * 64; }

static int64_t segment_slots(int rows, int num_seqs, int heads, int dv, int max_query_len) {
  const int per = segment_chunks(rows, heads, dv, max_query_len);
  if (max_query_len <= per * kChunk) return 0;
  return (int64_t)rows / (kChunk * per) + num_seqs + 1;
}

extern "C" int64_t lvllm_recurrent_mix_workspace_bytes(int rows, int num_seqs, int heads, int dk, int dv, int max_query_len) {
  if (max_query_len <= 1) return 0;
  const int64_t chunks = ((int64_t)rows / kChunk + num_seqs + 1) * heads * chunk_floats(padded_dk(dk));
  const int64_t segs = segment_slots(rows, num_seqs, heads, dv, max_query_len) * heads * ((int64_t)dk * dv + padded_dk(dk));
  return (chunks + 3 + segs) * 4;
}

extern "C" int lvllm_recurrent_mix(void* out, int64_t out_stride, const void* q, const void* k, const void* v,
                                   int64_t q_stride, int64_t k_stride, int64_t v_stride, const void* u, int64_t u_stride,
                                   const float* a_t, const float* decay_bias, int rank, int kind, float inv_tau,
                                   const float* bonus, float q_scale, const void* gate, int64_t gate_stride,
                                   const float* norm_weight, int norm_head_stride, float eps, float out_scale, float* state,
                                   int64_t state_stride, const int32_t* state_slots, int num_slots,
                                   const int32_t* query_start_loc, const int32_t* seq_lens, int num_seqs, int rows,
                                   int heads, int dk, int dv, int max_query_len, float* o_scratch, void* workspace,
                                   int64_t workspace_bytes, int dtype, void* stream) {
  if (num_seqs == 0 || rows == 0) return 0;
  LV_CHECK(dk > 0 && dk <= 256 && dv > 0 && dv <= 1024, "key size must be in 1 .. 256, value size in 1 .. 1024");
  LV_CHECK(kind == kDecayLogSigmoid || kind == kDecayNegExp, "unknown decay kind");
  LV_CHECK(rank > 0 && rank <= 1024, "rank must be in 1 .. 1024");
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
  LV_CHECK(workspace != nullptr && o_scratch != nullptr &&
               workspace_bytes >= lvllm_recurrent_mix_workspace_bytes(rows, num_seqs, heads, dk, dv, max_query_len),
           "workspace too small (see lvllm_recurrent_mix_workspace_bytes)");
  p.ws = (float*)workspace;
  p.o = o_scratch;
  p.seg_chunks = segment_chunks(rows, heads, dv, max_query_len);
  p.max_segs = (max_query_len + kChunk * p.seg_chunks - 1) / (kChunk * p.seg_chunks);
  LV_CHECK((int64_t)num_seqs * p.max_segs <= 65535, "too many sequences or too long portions");
  if (p.max_segs > 1) {  // (decays first: their rows are multiples of 16 bytes)
    p.seg_decay = p.ws + ((int64_t)rows / kChunk + num_seqs + 1) * heads * chunk_floats(padded_dk(dk));
    p.seg_state = p.seg_decay + segment_slots(rows, num_seqs, heads, dv, max_query_len) * heads * padded_dk(dk);
  }
  LV_DISPATCH_DTYPE(dtype, {
    switch (padded_dk(dk) / 64) {
      case 1: launch_chunks<scalar_t, 1>(p, rows, s); break;
      case 2: launch_chunks<scalar_t, 2>(p, rows, s); break;
      case 3: launch_chunks<scalar_t, 3>(p, rows, s); break;
      default: launch_chunks<scalar_t, 4>(p, rows, s); break;
    }
  });
  LV_LAUNCH_CHECK();
  return lvllm_head_norm_gate(out, out_stride, o_scratch, gate, gate_stride, norm_weight, norm_head_stride, eps, out_scale,
                              rows, heads, dv, dtype, stream);
}
