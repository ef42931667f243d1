// Linear recurrences with a matrix state per head and one decay per key channel, for gfx950:
//
//     S_t = diag(w_t) S_{t-1} + k_t v_t^T          S [dk, dv], fp32, carried per sequence
//     o_t = S_t^T q_t                              (plain read-out), or
//     o_t = (S_{t-1} + diag(u) k_t v_t^T)^T q_t    (bonus read-out: u weighs the current token)
//
// with low-rank data-dependent decays
//
//     z = A f(u_t) + bias,   ln w = logsigmoid(z) / tau   (f = identity)   or   ln w = -exp(z)   (f = tanh)
//
// (log_decay.h), or one fixed decay per head (FIXED), and then rotary positions on q and k, in fp32, where asked for.
//
// Two bodies:
//   * steps of single tokens (decode): ONE launch per mixer -- decay, state update, read-out, per-head RMS norm and gate --
//     a workgroup per (sequence, head) that streams the head's state through registers once: HBM-bound;
//   * everything else: the decays of all heads as one fp32-MFMA product (fixed decays: q and k rotated), then chunks of 16 tokens on fp32 MFMAs
//     (chunk_mix_kernel): per chunk the decay from its start is folded into q, the decay to its end into k; the masked
//     16 x 16 products inside the chunk, the read-out of the state before it and the state update are matrix products, the
//     per-head norm and gate its epilogue.  State tiles are MFMA accumulators AND, without a move, the B operands of the
//     read-out (k-step r of a tile contracts rows {r, 4 + r, 8 + r, 12 + r}: accumulator register r of every lane).
//     Sequences too few to fill the chip are cut into segments of chunks, whose states are found first.
//   Inside a chunk the decay between two tokens is the product of two factors measured from the chunk's middle; channels
//   that decay too fast for that (a factor would leave fp32's range) are left out and added pair by pair.
//
// QT is the element type of q and k: T, or fp32 where they were rotated.
// Everything but the projections' results (q, k, v, the low-rank input) is fp32: decays and their logarithms, the state,
// the read-out.  Rows are the new tokens of `num_seqs` sequences back to back (query_start_loc); a sequence whose tokens
// are all in this step (seq_lens == its rows) starts from a zero state, every other one from its slot.
#pragma once
#include "head_norm_gate.h"
#include "log_decay.h"
#include "rotation.h"
#include "row_ops.h"

namespace lvllm {

// ---- chunks of 16 tokens ------------------------------------------------------------------------------------------
struct MixParams {
  const void *q, *k, *v;  // row r, head h at r * stride + h * dk (dv)
  int64_t q_stride, k_stride, v_stride;
  const void* u;          // low-rank input, row stride u_stride
  int64_t u_stride;
  const float* a_t;       // [rank, heads * dk]
  const float* decay_bias;
  int kind, rank;
  float inv_tau;
  const float* head_decay;  // FIXED: [2, heads], the decays and their logarithms; low-rank decays otherwise
  const int64_t* positions; // FIXED, single tokens: [rows]; q and k are rotated
  const double* turns;      // [rot_dims / 2]
  int rot_dims;
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
  const float* norm_weight;  // null: none
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
template <typename T, typename QT, int NT, int NV, bool STATES, bool FIXED>
__global__ __launch_bounds__(256, NT == 1 && NV <= 4 ? 3 : 2) void chunk_mix_kernel(const MixParams p) {
  using S = typename T::store_t;
  using SQ = typename QT::store_t;
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
      nw[j] = !(epilogue && d0 + j < p.dv) ? 0.f
              : p.norm_weight == nullptr ? p.out_scale : p.norm_weight[head * p.norm_head_stride + d0 + j] * p.out_scale;
  }

  const float head_log = FIXED ? p.head_decay[p.heads + head] : 0.f;
  struct Frag {
    SQ q[NT][4], k[NT][4];
    float l[FIXED ? 1 : NT][4];
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
        if constexpr (!STATES) f.q[i][r] = ((const SQ*)p.q)[row * p.q_stride + ch];
        f.k[i][r] = ((const SQ*)p.k)[row * p.k_stride + ch];
        if constexpr (!FIXED) f.l[i][r] = p.log_decay[row * p.heads * p.dk + ch];
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
        if constexpr (FIXED) l[r] = 4 * g + r < nt ? head_log : 0.f;
        else l[r] = ok ? f.l[i][r] : 0.f;
        kv[r] = ok ? QT::to_float(f.k[i][r]) : 0.f;
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
          const float qv = t < nt && ch < p.dk ? QT::to_float(f.q[i][r]) * p.q_scale : 0.f;
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
              sq[t * LD + ch] = ok ? QT::to_float(((const SQ*)p.q)[row * p.q_stride + col]) * p.q_scale : 0.f;
              sk[t * LD + ch] = ok ? QT::to_float(((const SQ*)p.k)[row * p.k_stride + col]) : 0.f;
              if constexpr (FIXED) sl[t * LD + ch] = ok ? head_log : 0.f;
              else sl[t * LD + ch] = ok ? p.log_decay[row * p.heads * p.dk + col] : 0.f;
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
static __global__ __launch_bounds__(256) void chunk_combine_kernel(const MixParams p, const int dkp) {
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
template <typename T, int PRE, bool FIXED>
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
  const float u0 = FIXED ? 0.f : T::to_float(((const S*)p.u)[(int64_t)row * p.u_stride + min(tid, p.rank - 1)]);
  float q0 = T::to_float(((const S*)p.q)[(int64_t)row * p.q_stride + kc]) * p.q_scale;
  float k0 = T::to_float(((const S*)p.k)[(int64_t)row * p.k_stride + kc]);
  const float v0 = T::to_float(((const S*)p.v)[(int64_t)row * p.v_stride + vc]);
  const float gate0 = T::to_float(((const S*)p.gate)[(int64_t)row * p.gate_stride + vc]);
  const float weight0 = p.norm_weight != nullptr ? p.norm_weight[head * p.norm_head_stride + min(tid, dv - 1)] : 1.f;
  const float bias0 = FIXED ? 0.f : p.decay_bias[kc];
  const float bonus0 = p.bonus != nullptr ? p.bonus[kc] : 0.f;
  const float fixed0 = FIXED ? p.head_decay[head] : 0.f;
  float q1 = 0.f, k1 = 0.f;  // the other entry of a rotated pair
  double turns0 = 0.;
  const bool rotated = FIXED && tid < p.rot_dims;
  if (rotated) {
    const int half = p.rot_dims / 2, kc1 = head * dk + (tid < half ? tid + half : tid - half);
    q1 = T::to_float(((const S*)p.q)[(int64_t)row * p.q_stride + kc1]) * p.q_scale;
    k1 = T::to_float(((const S*)p.k)[(int64_t)row * p.k_stride + kc1]);
    turns0 = p.turns[tid < half ? tid : tid - half];
  }
  // z: the rank cut into parts, thread (part, channel)
  const int parts = FIXED ? 0 : 256 / dk, part_len = FIXED ? 0 : (p.rank + parts - 1) / parts;
  const int part = tid / dk, part_ch = tid - part * dk;
  const float* a = FIXED ? nullptr : p.a_t + head * dk + part_ch;
  const int64_t a_step = (int64_t)p.heads * dk;
  constexpr int AR = PRE == 4 ? 16 : 32;
  float a_pre[FIXED ? 1 : AR];
  if constexpr (!FIXED) {
#pragma unroll
    for (int i = 0; i < AR; ++i) a_pre[i] = a[min(part * part_len + i, p.rank - 1) * a_step];
  }
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
  if constexpr (!FIXED) {
    if (tid < p.rank) su[tid] = p.kind == kDecayNegExp ? tanhf(u0) : u0;
    for (int i = tid + 256; i < p.rank; i += 256) {
      const float f = T::to_float(((const S*)p.u)[(int64_t)row * p.u_stride + i]);
      su[i] = p.kind == kDecayNegExp ? tanhf(f) : f;
    }
  } else if (rotated) {
    float c, s;
    rotation_of(p.positions[row], turns0, c, s);
    const float sign = tid < p.rot_dims / 2 ? -s : s;
    q0 = q0 * c + q1 * sign;
    k0 = k0 * c + k1 * sign;
  }
  if (tid < dv) sv[tid] = v0;
  for (int i = tid + 256; i < dv; i += 256) sv[i] = T::to_float(((const S*)p.v)[(int64_t)row * p.v_stride + head * dv + i]);
  if (tid < dk) {
    sq[tid] = q0;
    sk[tid] = k0;
  }
  float bsum = 0.f;
  if constexpr (FIXED) {
    if (tid < dk) {
      sw[tid] = fixed0;
      bsum = q0 * bonus0 * k0;
    }
  } else {
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
    if (tid < dk) {
      float z = bias0;
      for (int q = 0; q < parts; ++q) z += so[q * dk + tid];
      sw[tid] = expf(log_decay_of(z, p.kind, p.inv_tau));
      bsum = q0 * bonus0 * k0;
    }
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
    const float w = first ? weight0 : p.norm_weight != nullptr ? p.norm_weight[head * p.norm_head_stride + d] : 1.f;
    const float silu = z / (1.f + expf(-z));
    ((S*)p.out)[(int64_t)row * p.out_stride + head * dv + d] = T::from_float(so[d] * r * w * silu * p.out_scale);
  }
}

// 64-channel groups of the state and 16-column tiles of a value slice
inline int key_groups(int dk) { return dk <= 64 ? 1 : dk <= 128 ? 2 : 4; }
inline int value_tiles(int dk, int dv) {
  const int most = dk <= 128 ? 8 : 4;
  int n = 1;
  while (n < most && n * 16 < dv) n *= 2;
  return n;
}
inline int value_slices(int dk, int dv) { return (dv + 16 * value_tiles(dk, dv) - 1) / (16 * value_tiles(dk, dv)); }

constexpr int mix_wgs_per_cu(int NT, int NV) { return NT == 1 && NV <= 4 ? 3 : 2; }  // (registers; the LDS holds as many)

// Chunks per segment: sequences are cut when (sequence, head, value slice) triples alone leave CUs idle, into as many
// segments as run at once
inline int segment_chunks(int rows, int heads, int dk, int dv, int max_query_len) {
  const int chunks = (max_query_len + kChunk - 1) / kChunk;
  const int64_t long_seqs = (rows + max_query_len - 1) / max_query_len;
  const int64_t wide = long_seqs * heads * value_slices(dk, dv);
  const int64_t segs = 256 * mix_wgs_per_cu(key_groups(dk), value_tiles(dk, dv)) / wide;
  const int per = segs < 2 ? chunks : (int)((chunks + segs - 1) / segs);
  return per < 8 ? 8 : per;
}
inline int64_t segment_slots(int rows, int num_seqs, int per, int max_query_len) {
  return max_query_len <= per * kChunk ? 0 : (int64_t)rows / (kChunk * per) + num_seqs + 1;
}

template <typename T, typename QT, int NT, int NV, bool FIXED>
static void launch_mix(const MixParams& p, hipStream_t s) {
  constexpr int smem = mix_smem_floats(NT, NV) * 4;
  const dim3 grid(p.heads, value_slices(p.dk, p.dv), p.num_seqs * p.max_segs);
  if (p.max_segs > 1) {
    hipLaunchKernelGGL((chunk_mix_kernel<T, QT, NT, NV, true, FIXED>), grid, dim3(256), 0, s, p);
    hipLaunchKernelGGL(chunk_combine_kernel, dim3((unsigned)(((int64_t)p.dk * p.dv + 255) / 256), p.heads, p.num_seqs),
                       dim3(256), 0, s, p, 64 * NT);
  }
  if (smem > 64 * 1024)
    (void)hipFuncSetAttribute((const void*)chunk_mix_kernel<T, QT, NT, NV, false, FIXED>, hipFuncAttributeMaxDynamicSharedMemorySize, smem);
  hipLaunchKernelGGL((chunk_mix_kernel<T, QT, NT, NV, false, FIXED>), grid, dim3(256), smem, s, p);
}

template <typename T, typename QT, bool FIXED>
static void launch_mix_sized(const MixParams& p, hipStream_t s) {
  const int nv = value_tiles(p.dk, p.dv);
  switch (key_groups(p.dk) * 16 + nv) {
    case 17: launch_mix<T, QT, 1, 1, FIXED>(p, s); break;
    case 18: launch_mix<T, QT, 1, 2, FIXED>(p, s); break;
    case 20: launch_mix<T, QT, 1, 4, FIXED>(p, s); break;
    case 24: launch_mix<T, QT, 1, 8, FIXED>(p, s); break;
    case 33: launch_mix<T, QT, 2, 1, FIXED>(p, s); break;
    case 34: launch_mix<T, QT, 2, 2, FIXED>(p, s); break;
    case 36: launch_mix<T, QT, 2, 4, FIXED>(p, s); break;
    case 40: launch_mix<T, QT, 2, 8, FIXED>(p, s); break;
    case 65: launch_mix<T, QT, 4, 1, FIXED>(p, s); break;
    case 66: launch_mix<T, QT, 4, 2, FIXED>(p, s); break;
    default: launch_mix<T, QT, 4, 4, FIXED>(p, s); break;
  }
}

// every sequence brings one token: sequence s owns row s
template <bool FIXED>
static int launch_single_tokens(const MixParams& p, int dtype, hipStream_t s) {
  const int dk = p.dk, dv = p.dv, cgs = (dv & 3) == 0 ? dv / 4 : dv, per = cgs < 256 ? cgs : 256, rgs = 256 / per;
  const int groups = rgs * dv > 256 ? rgs * dv : 256;
  const size_t smem = (size_t)(3 * dk + p.rank + 3 + dv + groups + 8) * sizeof(float);  // (at most 16 KB)
  const int pre = (dv & 3) == 0 ? (dk + rgs - 1) / rgs : 1 << 20;  // state rows per thread
  const dim3 grid(p.heads, p.num_seqs);
  LV_DISPATCH_F32_BF16(dtype, {
    if (pre <= 4) hipLaunchKernelGGL((recurrent_decode_kernel<scalar_t, 4, FIXED>), grid, dim3(256), smem, s, p);
    else if (pre <= 8) hipLaunchKernelGGL((recurrent_decode_kernel<scalar_t, 8, FIXED>), grid, dim3(256), smem, s, p);
    else if (pre <= 16) hipLaunchKernelGGL((recurrent_decode_kernel<scalar_t, 16, FIXED>), grid, dim3(256), smem, s, p);
    else hipLaunchKernelGGL((recurrent_decode_kernel<scalar_t, 0, FIXED>), grid, dim3(256), smem, s, p);
  });
  LV_LAUNCH_CHECK();
  return 0;
}

// The chunked body's segments; `ws`: their workspace.  Returns the floats taken.
inline int64_t plan_segments(MixParams& p, float* ws, int rows, int max_query_len) {
  p.seg_chunks = segment_chunks(rows, p.heads, p.dk, p.dv, max_query_len);
  p.max_segs = (max_query_len + kChunk * p.seg_chunks - 1) / (kChunk * p.seg_chunks);
  const int64_t segs = segment_slots(rows, p.num_seqs, p.seg_chunks, max_query_len) * p.heads;
  p.seg_decay = ws;
  p.seg_state = ws + segs * 64 * key_groups(p.dk);
  int64_t taken = segs * (64 * key_groups(p.dk) + (int64_t)p.dk * p.dv);
  if (value_slices(p.dk, p.dv) > 1) {
    p.o = ws + taken;
    taken += (int64_t)rows * p.heads * p.dv;
  }
  return taken;
}

inline int64_t segments_workspace(int rows, int num_seqs, int heads, int dk, int dv, int max_query_len) {  // floats
  const int per = segment_chunks(rows, heads, dk, dv, max_query_len);
  const int64_t segs = segment_slots(rows, num_seqs, per, max_query_len) * heads;
  const int64_t o = value_slices(dk, dv) > 1 ? (int64_t)rows * heads * dv : 0;
  return segs * ((int64_t)dk * dv + 64 * key_groups(dk)) + o;
}

}  // namespace lvllm
