// The gated delta rule (delta_rule.h).
#include "delta_rule.h"

#include "head_norm_gate.h"
#include "low_rank_decay.h"

namespace lvllm {

// state that is not touched again before the next step: past the caches
__device__ __forceinline__ r_f32x4_t load_past(const float* p) {
  return __builtin_nontemporal_load(reinterpret_cast<const r_f32x4_t*>(p));
}
__device__ __forceinline__ void store_past(float* p, r_f32x4_t v) {
  __builtin_nontemporal_store(v, reinterpret_cast<r_f32x4_t*>(p));
}

// The sums of three values over the workgroup; `red` is 48 floats.
__device__ __forceinline__ void block_sum3(float& a, float& b, float& c, float* red) {
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  a = wave_sum(a);
  b = wave_sum(b);
  c = wave_sum(c);
  if (lane == 0) {
    red[wave] = a;
    red[16 + wave] = b;
    red[32 + wave] = c;
  }
  __syncthreads();
  a = b = c = 0.f;
  for (int w = 0; w < (int)blockDim.x >> 6; ++w) {
    a += red[w];
    b += red[16 + w];
    c += red[32 + w];
  }
}

// ---- single tokens -------------------------------------------------------------------------------------------------
// LDS, in floats: what a workgroup keeps besides the reductions
struct StepLds {
  int k, w, u, z, v, gate, new_u, part_k, part_q, total;
  __host__ __device__ StepLds(int dk, int dv, int decay_rank, int gate_rank, int groups) {
    auto up = [](int n) { return (n + 7) & ~7; };
    k = up(dk);
    w = k + up(dk);
    u = w + up(dk);
    z = u + up(decay_rank);
    v = z + up(gate_rank);
    gate = v + up(dv);
    new_u = gate + up(dv);
    part_k = new_u + up(dv);
    part_q = part_k + up(groups * dv);
    total = part_q + up(groups * dv);
  }
};
// threads along a state row, in columns of VEC, and rows at once
__host__ __device__ inline int step_columns(int dv, int vec) { return dv / vec < 256 ? dv / vec : 256; }

// PRE > 0: a thread's PRE state rows are loaded before anything is computed and stay in registers; 0: any size, two passes over
// memory.  Thread (rg, cg): columns VEC cg .. of rows rg, rg + RG, ...
template <typename T, int PRE, int VEC>
__global__ __launch_bounds__(256) void delta_step_kernel(const DeltaStepParams p) {
  using S = typename T::store_t;
  constexpr int X = 16 / sizeof(S);
  constexpr int NP = PRE == 16 ? 8 : 16;  // pieces of low-rank weights asked for ahead of the state
  constexpr int kAhead = 4;               // taps held in registers
  extern __shared__ __attribute__((aligned(16))) float sm[];
  __shared__ float red[48];
  const int head = blockIdx.x, seq = blockIdx.y, tid = threadIdx.x;
  const int dk = p.dk, dv = p.dv;
  const int per = step_columns(dv, VEC), rgs = 256 / per, rg = tid / per, cg0 = tid - rg * per, cgs = dv / VEC;
  const StepLds lds(dk, dv, p.decay_rank, p.gate_rank, rgs);
  float *sq = sm, *sk = sm + lds.k, *sw = sm + lds.w, *su = sm + lds.u, *sz = sm + lds.z, *sv = sm + lds.v;
  float *sgate = sm + lds.gate, *snew = sm + lds.new_u, *spk = sm + lds.part_k, *spq = sm + lds.part_q;
  const int group = p.heads / p.kv_heads, qc = head / group * dk;
  const int slot = p.state_slots[seq];
  const bool live = slot >= 0 && slot < p.num_slots;
  const int pos = max(p.seq_lens[seq] - 1, 0);
  const bool fresh = pos == 0 || !live;
  float* st = p.state + (int64_t)(live ? slot : 0) * p.state_stride + (int64_t)head * dk * dv;
  float* ring = p.conv_state + (int64_t)(live ? slot : 0) * p.conv_stride;
  const int64_t at = seq * p.x_stride;  // (sequence s owns row s)
  const S* x = (const S*)p.x + at;
  const int ring_row = pos % p.taps;

  // Loads return in order: the small operands first, the state behind them.
  struct Channel {
    float now, w[kAhead], old[kAhead];
  };
  auto ask = [&](int c, Channel& h) __attribute__((always_inline)) {
    h.now = T::to_float(x[c]);
#pragma unroll
    for (int j = 0; j < kAhead; ++j) {
      h.w[j] = h.old[j] = 0.f;
      if (j >= p.taps) continue;
      h.w[j] = p.conv_weight[(int64_t)(p.taps - 1 - j) * p.channels + c];
      const int r = ring_row - j;
      if (j > 0 && j <= pos && live) h.old[j] = ring[(int64_t)(r < 0 ? r + p.taps : r) * p.channels + c];
    }
  };
  auto convolve = [&](int c, const Channel& h, bool keep) __attribute__((always_inline)) {
    float y = h.now * h.w[0];
#pragma unroll
    for (int j = 1; j < kAhead; ++j) y = fmaf(h.w[j], h.old[j], y);
    for (int j = kAhead; j < p.taps && j <= pos && live; ++j) {
      const int r = ring_row - j;
      const float old = ring[(int64_t)(r < 0 ? r + p.taps : r) * p.channels + c];
      y = fmaf(p.conv_weight[(int64_t)(p.taps - 1 - j) * p.channels + c], old, y);
    }
    if (keep && live) ring[(int64_t)ring_row * p.channels + c] = h.now;  // (read by nobody in this step)
    return silu_of(y);
  };
  Channel cq, ck, cv;
  const int kc = min(tid, dk - 1), vc = min(tid, dv - 1);
  ask(qc + kc, cq);
  ask(p.k_at + qc + kc, ck);
  ask(p.v_at + head * dv + vc, cv);
  const float beta = 1.f / (1.f + expf(-T::to_float(((const S*)p.beta)[at + head])));
  const int cols = dk + dv;
  auto weights_of = [&](int col, const S*& w, int64_t& step, int& pieces, const float*& in) __attribute__((always_inline)) {
    const bool decay = col < dk;
    w = decay ? (const S*)p.decay_w + ((int64_t)head * dk + col) * X : (const S*)p.gate_w + ((int64_t)head * dv + col - dk) * X;
    step = (int64_t)p.heads * (decay ? dk : dv) * X;
    pieces = ((decay ? p.decay_rank : p.gate_rank) + X - 1) / X;
    in = decay ? su : sz;
  };
  const S* w0;
  const float* in0;
  int64_t step0;
  int pieces0;
  weights_of(min(tid, cols - 1), w0, step0, pieces0, in0);
  Vec16<T> ahead[NP];
#pragma unroll
  for (int i = 0; i < NP; ++i) ahead[i] = *reinterpret_cast<const Vec16<T>*>(w0 + min(i, pieces0 - 1) * step0);
  const float scale0 = p.decay_scale[head * dk + kc], bias0 = p.decay_bias[head * dk + kc], norm0 = p.norm_weight[vc];
  for (int i = tid; i < lds.z - lds.u; i += 256) su[i] = i < p.decay_rank ? T::to_float(((const S*)p.u)[at + i]) : 0.f;
  for (int i = tid; i < lds.v - lds.z; i += 256) sz[i] = i < p.gate_rank ? T::to_float(((const S*)p.z)[at + i]) : 0.f;
  r_f32x4_t pre[PRE > 0 ? PRE : 1];
  if constexpr (PRE > 0) {
#pragma unroll
    for (int i = 0; i < PRE; ++i) {
      pre[i] = r_f32x4_t{0.f, 0.f, 0.f, 0.f};
      const int r = rg + i * rgs;
      if (!fresh && rg < rgs && r < dk) pre[i] = load_past(st + (int64_t)r * dv + 4 * cg0);
    }
  }
  // convolutions (raw q and k go to LDS, their lengths are put in where they are used)
  const bool keeps = head % group == 0;
  const float q = convolve(qc + kc, cq, keeps && tid < dk), k = convolve(p.k_at + qc + kc, ck, keeps && tid < dk);
  const float v0 = convolve(p.v_at + head * dv + vc, cv, tid < dv);
  if (tid < dk) {
    sq[tid] = q;
    sk[tid] = k;
  }
  if (tid < dv) sv[tid] = v0;
  for (int d = tid + 256; d < dv; d += 256) {
    Channel h;
    ask(p.v_at + head * dv + d, h);
    sv[d] = convolve(p.v_at + head * dv + d, h, true);
  }
  __syncthreads();
  auto take = [&](int col, float sum) __attribute__((always_inline)) {
    if (col < dk) {
      const bool first = col == tid;
      const int c = head * dk + col;
      sw[col] = exp_of(log_decay_of(sum + (first ? bias0 : p.decay_bias[c]), kDecaySoftplus, first ? scale0 : p.decay_scale[c]));
    } else {
      sgate[col - dk] = 1.f / (1.f + expf(-sum));
    }
  };
  for (int col = tid; col < cols; col += 256) {
    const S* w = w0;
    const float* in = in0;
    int64_t step = step0;
    int pieces = pieces0, i0 = 0;
    float sum = 0.f;
    if (col == tid) {
#pragma unroll
      for (int i = 0; i < NP; ++i)
        if (i < pieces) {
#pragma unroll
          for (int j = 0; j < X; ++j) sum = fmaf(in[i * X + j], T::to_float(ahead[i].v[j]), sum);
        }
      i0 = NP;
    } else {
      weights_of(col, w, step, pieces, in);
    }
#pragma unroll 4
    for (int i = i0; i < pieces; ++i) {
      const Vec16<T> t = *reinterpret_cast<const Vec16<T>*>(w + i * step);
#pragma unroll
      for (int j = 0; j < X; ++j) sum = fmaf(in[i * X + j], T::to_float(t.v[j]), sum);
    }
    take(col, sum);
  }
  float qq = tid < dk ? q * q : 0.f, kk = tid < dk ? k * k : 0.f, kq = tid < dk ? k * q : 0.f;
  block_sum3(qq, kk, kq, red);  // (a barrier: decays and gates are visible behind it)
  const float fk = 1.f / sqrtf(kk + kUnitEps), fq = p.q_scale / sqrtf(qq + kUnitEps);
  // w = diag(g) S, and its products with k and q
  if constexpr (PRE > 0) {
    if (rg < rgs) {
      r_f32x4_t ak{0.f, 0.f, 0.f, 0.f}, aq{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int i = 0; i < PRE; ++i) {
        const int r = rg + i * rgs;
        if (r < dk) {
          const float g = sw[r], kr = sk[r], qr = sq[r];
#pragma unroll
          for (int j = 0; j < 4; ++j) {
            pre[i][j] *= g;
            ak[j] = fmaf(kr, pre[i][j], ak[j]);
            aq[j] = fmaf(qr, pre[i][j], aq[j]);
          }
        }
      }
      *reinterpret_cast<r_f32x4_t*>(spk + rg * dv + 4 * cg0) = ak;
      *reinterpret_cast<r_f32x4_t*>(spq + rg * dv + 4 * cg0) = aq;
    }
  } else if (rg < rgs) {
    for (int cg = cg0; cg < cgs; cg += per) {
      float ak[VEC], aq[VEC];
#pragma unroll
      for (int j = 0; j < VEC; ++j) ak[j] = aq[j] = 0.f;
      for (int r = rg; r < dk && !fresh; r += rgs) {
        const float g = sw[r], kr = sk[r], qr = sq[r];
#pragma unroll
        for (int j = 0; j < VEC; ++j) {
          const float n = g * st[(int64_t)r * dv + VEC * cg + j];
          ak[j] = fmaf(kr, n, ak[j]);
          aq[j] = fmaf(qr, n, aq[j]);
        }
      }
#pragma unroll
      for (int j = 0; j < VEC; ++j) {
        spk[rg * dv + VEC * cg + j] = ak[j];
        spq[rg * dv + VEC * cg + j] = aq[j];
      }
    }
  }
  __syncthreads();
  float ss = 0.f;
  for (int d = tid; d < dv; d += 256) {
    float ak = 0.f, aq = 0.f;
    for (int r = 0; r < rgs; ++r) {
      ak += spk[r * dv + d];
      aq += spq[r * dv + d];
    }
    const float u = beta * (sv[d] - fk * ak), o = fmaf(kq * fk * fq, u, fq * aq);
    snew[d] = fk * u;
    spq[d] = o;  // (column d is this thread's alone)
    ss = fmaf(o, o, ss);
  }
  const float f = 1.f / sqrtf(block_sum(ss, red) / dv + p.eps);  // (barriers: the new u is visible behind them)
  if (live) {
    if constexpr (PRE > 0) {
      if (rg < rgs) {
        const r_f32x4_t u = *reinterpret_cast<const r_f32x4_t*>(snew + 4 * cg0);
#pragma unroll
        for (int i = 0; i < PRE; ++i) {
          const int r = rg + i * rgs;
          if (r < dk) {
            const float kr = sk[r];
            r_f32x4_t n;
#pragma unroll
            for (int j = 0; j < 4; ++j) n[j] = fmaf(kr, u[j], pre[i][j]);
            store_past(st + (int64_t)r * dv + 4 * cg0, n);
          }
        }
      }
    } else if (rg < rgs) {
      for (int cg = cg0; cg < cgs; cg += per)
        for (int r = rg; r < dk; r += rgs) {
          float* s = st + (int64_t)r * dv + VEC * cg;
          const float g = sw[r], kr = sk[r];
#pragma unroll
          for (int j = 0; j < VEC; ++j) s[j] = fmaf(kr, snew[VEC * cg + j], fresh ? 0.f : g * s[j]);
        }
    }
  }
  S* out = (S*)p.out + seq * p.out_stride + (int64_t)head * dv;
  for (int d = tid; d < dv; d += 256)
    out[d] = T::from_float(spq[d] * f * (d == tid ? norm0 : p.norm_weight[d]) * sgate[d]);
}

// ---- chunks --------------------------------------------------------------------------------------------------------
__host__ __device__ constexpr int prepare_lds_floats(int NT) {
  return 5 * kChunk * (64 * NT + 4) + 8 * 256 + kChunk * (kChunk + 4) + 8 * kChunk + kChunk + 4 * NT;
}

// One workgroup per (head, chunk).  Wave w owns key channels [16 NT w, 16 NT (w + 1)); a lane loads channel c, tokens 4g .. 4g + 3
// of a tile.  Channels that decay too fast for two factors measured from the chunk's middle are added pair by pair.
template <typename T, int NT>
__global__ __launch_bounds__(256, NT <= 2 ? 2 : 1) void delta_prepare_kernel(const DeltaChunkParams p) {
  using S = typename T::store_t;
  constexpr int DKP = 64 * NT, LD = DKP + 4, LA = kChunk + 4;
  extern __shared__ __attribute__((aligned(16))) float sm[];
  float* sq = sm;                   // [16][LD]: q from the middle of the chunk
  float* sk = sq + kChunk * LD;     // [16][LD]: k to the middle
  float* sr = sk + kChunk * LD;     // [16][LD]: k from the middle (fast decays: ln g)
  float* sqs = sr + kChunk * LD;    // [16][LD]: q from the chunk's start
  float* sks = sqs + kChunk * LD;   // [16][LD]: beta k from the chunk's start, then W
  float* spart = sks + kChunk * LD;  // [2][4 waves][16][16]: products of q and of k with k
  float* sa = spart + 8 * 256;      // [16][LA]: the system's matrix below its diagonal
  float* sn = sa + kChunk * LA;     // [2][4 waves][16]: squares
  float* sb = sn + 8 * kChunk;      // [16]: beta
  int* swild = reinterpret_cast<int*>(sb + kChunk);  // [4 NT]: channels of a tile that decay too fast
  const int head = blockIdx.x, slot = blockIdx.y;
  int seq = 0;
  for (int n = p.num_seqs; n > 1;) {  // the last sequence that begins at or before this slot
    const int half = n >> 1;
    if (chunk_slot_base(p.query_start_loc, seq + half) <= slot) {
      seq += half;
      n -= half;
    } else {
      n = half;
    }
  }
  const int ci = slot - chunk_slot_base(p.query_start_loc, seq);
  const int qbeg = p.query_start_loc[seq], qlen = p.query_start_loc[seq + 1] - qbeg;
  if (ci < 0 || ci * kChunk >= qlen) return;
  const int nt = min(kChunk, qlen - ci * kChunk);
  const int lane = threadIdx.x & 63;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int g = lane >> 4, c = lane & 15;
  const int dk = p.dk, dv = p.dv, qc = head / (p.heads / p.kv_heads) * dk;
  float* ws = p.chunks + ((int64_t)slot * p.heads + head) * p.layout.size();
  const S* y = (const S*)p.y;
  auto row_of = [&](int t) { return (int64_t)(qbeg + min(ci * kChunk + t, qlen - 1)); };
  float qv[NT][4], kv[NT][4], lv[NT][4];
  float qq[4], kk[4];
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int64_t row = row_of(4 * g + r);
    qq[r] = kk[r] = 0.f;
#pragma unroll
    for (int i = 0; i < NT; ++i) {
      const int ch = (wave * NT + i) * 16 + c, cc = min(ch, dk - 1);
      const bool ok = 4 * g + r < nt && ch < dk;
      const float a = T::to_float(y[row * p.y_stride + qc + cc]), b = T::to_float(y[row * p.y_stride + p.k_at + qc + cc]);
      const float l = p.log_decay[(row * p.heads + head) * dk + cc];
      qv[i][r] = ok ? a : 0.f;
      kv[i][r] = ok ? b : 0.f;
      lv[i][r] = ok ? l : 0.f;
      qq[r] = fmaf(qv[i][r], qv[i][r], qq[r]);
      kk[r] = fmaf(kv[i][r], kv[i][r], kk[r]);
    }
  }
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    qq[r] = group_sum<16>(qq[r]);
    kk[r] = group_sum<16>(kk[r]);
    if (c == 0) {
      sn[wave * 16 + 4 * g + r] = qq[r];
      sn[64 + wave * 16 + 4 * g + r] = kk[r];
    }
  }
  if (threadIdx.x < kChunk) {
    const float z = T::to_float(((const S*)p.beta)[row_of(threadIdx.x) * p.beta_stride + head]);
    sb[threadIdx.x] = 1.f / (1.f + expf(-z));
  }
  __syncthreads();
  float beta[4];
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int t = 4 * g + r;
    const float fq = p.q_scale / sqrtf(((sn[t] + sn[16 + t]) + (sn[32 + t] + sn[48 + t])) + kUnitEps);
    const float fk = 1.f / sqrtf(((sn[64 + t] + sn[80 + t]) + (sn[96 + t] + sn[112 + t])) + kUnitEps);
    beta[r] = sb[t];
#pragma unroll
    for (int i = 0; i < NT; ++i) {
      qv[i][r] *= fq;
      kv[i][r] *= fk;
    }
  }
  bool wild = false;
#pragma unroll
  for (int i = 0; i < NT; ++i) {
    const int tile = wave * NT + i, ch = tile * 16 + c;
    const ChunkSums cs(lv[i], g, c, false);
    const bool mild = -cs.h1 < kMaxHalfDecay && -cs.h2 < kMaxHalfDecay;
    wild = wild || !mild;
    const uint64_t fast = __ballot(!mild);
    if (lane == 0) swild[tile] = (int)(fast & 0xffff);
    const float to_mid = exp_of(cs.h1), from_mid = exp_of(cs.h2);
    float kend[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int t = 4 * g + r;
      const float from = mild ? exp_of(cs.half_q[r]) : 0.f, to = mild ? exp_of(cs.half_k[r]) : 0.f;
      const float read = mild ? from * to_mid : exp_of(cs.read[r]);
      sq[t * LD + ch] = qv[i][r] * from;
      sr[t * LD + ch] = kv[i][r] * from;
      sk[t * LD + ch] = kv[i][r] * to;
      sqs[t * LD + ch] = qv[i][r] * read;
      sks[t * LD + ch] = beta[r] * kv[i][r] * read;
      kend[r] = kv[i][r] * (mild ? to * from_mid : exp_of(cs.left[r]));
    }
    *reinterpret_cast<float4*>(ws + p.layout.k() + (tile * 64 + lane) * 4) = float4{kend[0], kend[1], kend[2], kend[3]};
    if (g == 0) ws[p.layout.end() + ch] = exp_of(cs.h1 + cs.h2);
  }
  // this wave's channels only: what it wrote itself, no barrier needed
  __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
  __builtin_amdgcn_wave_barrier();
  {
    r_f32x4_t pq{0.f, 0.f, 0.f, 0.f}, pk{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int i = 0; i < NT; ++i) {
      const int ch0 = (wave * NT + i) * 16 + 4 * g;
      const float4 a = *reinterpret_cast<const float4*>(sq + c * LD + ch0), b = *reinterpret_cast<const float4*>(sr + c * LD + ch0);
      const float4 k = *reinterpret_cast<const float4*>(sk + c * LD + ch0);
      pq = mfma_f32(a.x, k.x, pq); pk = mfma_f32(b.x, k.x, pk);
      pq = mfma_f32(a.y, k.y, pq); pk = mfma_f32(b.y, k.y, pk);
      pq = mfma_f32(a.z, k.z, pq); pk = mfma_f32(b.z, k.z, pk);
      pq = mfma_f32(a.w, k.w, pq); pk = mfma_f32(b.w, k.w, pk);
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      spart[wave * 256 + (4 * g + r) * 16 + c] = pq[r];
      spart[1024 + wave * 256 + (4 * g + r) * 16 + c] = pk[r];
    }
  }
  const int ti = threadIdx.x >> 4, tj = threadIdx.x & 15;
  float extra_q = 0.f, extra_k = 0.f;
  if (__syncthreads_or(wild)) {  // the products of the channels left out above
#pragma unroll
    for (int i = 0; i < NT; ++i) {
      const int ch = (wave * NT + i) * 16 + c;
      if (swild[wave * NT + i] >> c & 1) {
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int t = 4 * g + r;
          sq[t * LD + ch] = qv[i][r];
          sk[t * LD + ch] = kv[i][r];
          sr[t * LD + ch] = lv[i][r];
        }
      }
    }
    __syncthreads();
    if (tj <= ti) {
      for (int i = 0; i < 4 * NT; ++i)
        for (int left = swild[i]; left != 0; left &= left - 1) {
          const int ch = i * 16 + __builtin_ctz(left);
          float between = 0.f;
          for (int t = tj + 1; t <= ti; ++t) between += sr[t * LD + ch];
          const float k = sk[tj * LD + ch] * exp_of(between);
          extra_q = fmaf(sq[ti * LD + ch], k, extra_q);
          extra_k = fmaf(sk[ti * LD + ch], k, extra_k);
        }
    }
  }
  {
    const int at = threadIdx.x;  // token ti, token tj
    const float pq = (spart[at] + spart[256 + at]) + (spart[512 + at] + spart[768 + at]) + extra_q;
    const float pk = (spart[1024 + at] + spart[1280 + at]) + (spart[1536 + at] + spart[1792 + at]) + extra_k;
    ws[p.layout.p() + (tj & 3) * 64 + (tj >> 2) * 16 + ti] = tj <= ti ? pq : 0.f;
    sa[ti * LA + tj] = tj < ti ? sb[ti] * pk : 0.f;
  }
  __syncthreads();
  // substitution: a thread per column of beta G k and of beta v
  for (int col = threadIdx.x; col < DKP + p.layout.dvp; col += 256) {
    const int d = col - DKP;
    float x[16];
    if (d < 0) {
      if (col >= dk) continue;  // (zeros already)
#pragma unroll
      for (int t = 0; t < 16; ++t) x[t] = sks[t * LD + col];
    } else {
      const int dc = p.v_at + head * dv + min(d, dv - 1);
#pragma unroll
      for (int t = 0; t < 16; ++t) {
        const float v = T::to_float(y[row_of(t) * p.y_stride + dc]);
        x[t] = t < nt && d < dv ? v * sb[t] : 0.f;
      }
    }
#pragma unroll
    for (int t = 1; t < 16; ++t) {
      float4 a[4];
#pragma unroll
      for (int j = 0; j < (t + 3) / 4; ++j) a[j] = *reinterpret_cast<const float4*>(sa + t * LA + 4 * j);
#pragma unroll
      for (int j = 0; j < (t + 3) / 4; ++j) {
        x[t] = fmaf(-a[j].x, x[4 * j], x[t]);
        if (4 * j + 1 < t) x[t] = fmaf(-a[j].y, x[4 * j + 1], x[t]);
        if (4 * j + 2 < t) x[t] = fmaf(-a[j].z, x[4 * j + 2], x[t]);
        if (4 * j + 3 < t) x[t] = fmaf(-a[j].w, x[4 * j + 3], x[t]);
      }
    }
    if (d < 0) {
#pragma unroll
      for (int t = 0; t < 16; ++t) sks[t * LD + col] = x[t];
    } else {
      float* u = ws + p.layout.u() + (d >> 4) * 256 + (d & 15);
#pragma unroll
      for (int t = 0; t < 16; ++t) u[(t & 3) * 64 + (t >> 2) * 16] = x[t];
    }
  }
  __syncthreads();
#pragma unroll
  for (int i = 0; i < NT; ++i) {
    const int tile = wave * NT + i, from = c * LD + tile * 16 + 4 * g, to = (tile * 64 + lane) * 4;
    *reinterpret_cast<float4*>(ws + p.layout.w() + to) = *reinterpret_cast<const float4*>(sks + from);
    *reinterpret_cast<float4*>(ws + p.layout.q() + to) = *reinterpret_cast<const float4*>(sqs + from);
  }
}

// everything written to LDS so far is seen by the workgroup; loads in flight stay in flight
__device__ __forceinline__ void delta_barrier() { asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory"); }

// One workgroup per (head, slice of 16 NV value columns, sequence).  State tiles are accumulators that serve as B operands
// unmoved (k-step r of a tile contracts its rows r, 4 + r, 8 + r, 12 + r); so is u.
template <int NT, int NV>
__global__ __launch_bounds__(256, NT * NV <= 4 ? 2 : 1) void delta_scan_kernel(const DeltaChunkParams p) {
  __shared__ __attribute__((aligned(16))) float swu[2][4][NV][256], so[2][4][NV][256];
  const int head = blockIdx.x, seq = blockIdx.z, tile0 = blockIdx.y * NV, tiles = p.layout.dvp >> 4;
  const int qbeg = p.query_start_loc[seq], qlen = p.query_start_loc[seq + 1] - qbeg;
  if (qlen <= 0) return;
  const int chunks = (qlen + kChunk - 1) / kChunk;
  const int lane = threadIdx.x & 63;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int g = lane >> 4, c = lane & 15;
  const int slot = p.state_slots[seq], dk = p.dk, dv = p.dv;
  const bool live = slot >= 0 && slot < p.num_slots, fresh = !live || p.seq_lens[seq] <= qlen;
  float* st = p.state + (int64_t)(live ? slot : 0) * p.state_stride + (int64_t)head * dk * dv;
  r_f32x4_t s[NT][NV];
#pragma unroll
  for (int i = 0; i < NT; ++i)
#pragma unroll
    for (int j = 0; j < NV; ++j)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int row = (wave * NT + i) * 16 + 4 * g + r, col = (tile0 + j) * 16 + c;
        s[i][j][r] = !fresh && row < dk && col < dv ? st[(int64_t)row * dv + col] : 0.f;
      }
  const int64_t step = (int64_t)p.heads * p.layout.size();
  const float* ws = p.chunks + ((int64_t)chunk_slot_base(p.query_start_loc, seq) * p.heads + head) * p.layout.size();
  struct Frag {
    float4 w[NT], q[NT], k[NT], end[NT];
    float u[NV], pr;  // this wave's rows 4 g + wave of U, and columns 4 g + wave of P
  };
  const int tile_at = wave * NT * 256 + lane * 4;
  auto load_tiles = [&](int ci, int piece, float4 (&to)[NT]) __attribute__((always_inline)) {
    const float* at = ws + min(ci, chunks - 1) * step + piece + tile_at;
#pragma unroll
    for (int i = 0; i < NT; ++i) to[i] = *reinterpret_cast<const float4*>(at + i * 256);
  };
  auto load_rest = [&](int ci, Frag& f) __attribute__((always_inline)) {
    const float* at = ws + min(ci, chunks - 1) * step;
#pragma unroll
    for (int i = 0; i < NT; ++i) f.end[i] = *reinterpret_cast<const float4*>(at + p.layout.end() + (wave * NT + i) * 16 + 4 * g);
#pragma unroll
    for (int j = 0; j < NV; ++j) f.u[j] = at[p.layout.u() + min(tile0 + j, tiles - 1) * 256 + wave * 64 + lane];
    f.pr = at[p.layout.p() + wave * 64 + lane];
  };
  // (conditions per lane: selects, no branches)
  const bool odd_wave = (threadIdx.x >> 6) & 1, high_wave = (threadIdx.x >> 7) & 1;
  auto of_wave = [&](float x, float y, float z, float w) {
    const float lo = odd_wave ? y : x, hi = odd_wave ? w : z;
    return high_wave ? hi : lo;
  };
  // token et, column ec of a tile: where the accumulator layout has it
  const int et = threadIdx.x >> 4, ec = threadIdx.x & 15, eat = ((et >> 2) * 16 + ec) * 4 + (et & 3);
  float* out = p.o + ((int64_t)(qbeg + et) * p.heads + head) * dv + tile0 * 16 + ec;  // of the chunk read out next
  const int64_t out_step = (int64_t)kChunk * p.heads * dv;
  auto read_out = [&](int ci, const float (&o)[NV][4]) __attribute__((always_inline)) {
#pragma unroll
    for (int j = 0; j < NV; ++j)
      if (ci * kChunk + et < qlen && (tile0 + j) * 16 + ec < dv) out[16 * j] = (o[j][0] + o[j][1]) + (o[j][2] + o[j][3]);
    out += out_step;
  };
  auto shares_of = [&](int par, float (&o)[NV][4]) __attribute__((always_inline)) {
#pragma unroll
    for (int j = 0; j < NV; ++j)
#pragma unroll
      for (int w = 0; w < 4; ++w) o[j][w] = so[par][w][j][eat];
  };
  // par: ci & 1.  The waves' shares of W S - U meet in LDS; half of (G q) S is computed while they are written, half while they
  // are read.  What a later chunk needs is asked for as soon as its registers are free.
  auto chunk = [&](int ci, int ahead, int par, Frag& f) __attribute__((always_inline)) {
    r_f32x4_t a[NV], o[NV];
    auto times_state = [&](int j, const float4 (&x)[NT], int r, r_f32x4_t acc) __attribute__((always_inline)) {
#pragma unroll
      for (int i = 0; i < NT; ++i)
        acc = mfma_f32(r == 0 ? x[i].x : r == 1 ? x[i].y : r == 2 ? x[i].z : x[i].w, s[i][j][r], acc);
      return acc;
    };
#pragma unroll
    for (int j = 0; j < NV; ++j) {
      const float u = -f.u[j];
      a[j] = r_f32x4_t{odd_wave || high_wave ? 0.f : u, !odd_wave || high_wave ? 0.f : u, odd_wave || !high_wave ? 0.f : u,
                       odd_wave && high_wave ? u : 0.f};
      o[j] = r_f32x4_t{0.f, 0.f, 0.f, 0.f};
    }
#pragma unroll
    for (int r = 0; r < 4; ++r)
#pragma unroll
      for (int j = 0; j < NV; ++j) a[j] = times_state(j, f.w, r, a[j]);
#pragma unroll
    for (int j = 0; j < NV; ++j) o[j] = times_state(j, f.q, 0, o[j]);
    __builtin_amdgcn_sched_barrier(0);
    load_tiles(ci + ahead, p.layout.w(), f.w);
#pragma unroll
    for (int j = 0; j < NV; ++j) *reinterpret_cast<r_f32x4_t*>(&swu[par][wave][j][lane * 4]) = a[j];
#pragma unroll
    for (int j = 0; j < NV; ++j) o[j] = times_state(j, f.q, 1, o[j]);
    __builtin_amdgcn_sched_barrier(0);
    delta_barrier();
    r_f32x4_t t[NV][4];
    float before[NV][4];  // the chunk before's read-out is complete
#pragma unroll
    for (int j = 0; j < NV; ++j)
#pragma unroll
      for (int w = 0; w < 4; ++w) t[j][w] = *reinterpret_cast<const r_f32x4_t*>(&swu[par][w][j][lane * 4]);
    shares_of(par ^ 1, before);
    __builtin_amdgcn_sched_barrier(0);
#pragma unroll
    for (int r = 2; r < 4; ++r)
#pragma unroll
      for (int j = 0; j < NV; ++j) o[j] = times_state(j, f.q, r, o[j]);
#pragma unroll
    for (int i = 0; i < NT; ++i)
#pragma unroll
      for (int j = 0; j < NV; ++j) {
        s[i][j][0] *= f.end[i].x; s[i][j][1] *= f.end[i].y; s[i][j][2] *= f.end[i].z; s[i][j][3] *= f.end[i].w;
      }
    __builtin_amdgcn_sched_barrier(0);
    load_tiles(ci + ahead, p.layout.q(), f.q);
    const float pr = f.pr;
    load_rest(ci + ahead, f);
#pragma unroll
    for (int j = 0; j < NV; ++j) {
      r_f32x4_t u;
#pragma unroll
      for (int r = 0; r < 4; ++r) u[r] = -((t[j][0][r] + t[j][1][r]) + (t[j][2][r] + t[j][3][r]));
      o[j] = mfma_f32(pr, of_wave(u[0], u[1], u[2], u[3]), o[j]);
#pragma unroll
      for (int r = 0; r < 4; ++r)
#pragma unroll
        for (int i = 0; i < NT; ++i)
          s[i][j] = mfma_f32(r == 0 ? f.k[i].x : r == 1 ? f.k[i].y : r == 2 ? f.k[i].z : f.k[i].w, u[r], s[i][j]);
    }
    __builtin_amdgcn_sched_barrier(0);
    load_tiles(ci + ahead, p.layout.k(), f.k);
    if (ci > 0) read_out(ci - 1, before);
#pragma unroll
    for (int j = 0; j < NV; ++j) *reinterpret_cast<r_f32x4_t*>(&so[par][wave][j][lane * 4]) = o[j];
  };
  constexpr int kDepth = NT * NV <= 2 ? 4 : 2;  // chunks asked for ahead
  Frag f[kDepth];
#pragma unroll
  for (int d = 0; d < kDepth; ++d) {
    load_tiles(d, p.layout.w(), f[d].w);
    load_tiles(d, p.layout.q(), f[d].q);
    load_rest(d, f[d]);
    load_tiles(d, p.layout.k(), f[d].k);
  }
  for (int ci = 0; ci < chunks; ci += kDepth) {
#pragma unroll
    for (int d = 0; d < kDepth; ++d)
      if (ci + d < chunks) chunk(ci + d, kDepth, d & 1, f[d]);
  }
  delta_barrier();
  float last[NV][4];
  shares_of((chunks - 1) & 1, last);
  read_out(chunks - 1, last);
  if (!live) return;
#pragma unroll
  for (int i = 0; i < NT; ++i)
#pragma unroll
    for (int j = 0; j < NV; ++j)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int row = (wave * NT + i) * 16 + 4 * g + r, col = (tile0 + j) * 16 + c;
        if (row < dk && col < dv) st[(int64_t)row * dv + col] = s[i][j][r];
      }
}

static int key_tiles(int dk) { return dk <= 64 ? 1 : dk <= 128 ? 2 : 4; }
static ChunkLayout chunk_layout(int dk, int dv) { return ChunkLayout{64 * key_tiles(dk), (dv + 15) / 16 * 16}; }

template <int NT>
static int launch_scan(const DeltaChunkParams& p, int rows, int max_query_len, hipStream_t s) {
  const int tiles = p.layout.dvp / 16;
  const int64_t wide = (int64_t)((rows + max_query_len - 1) / max_query_len) * p.heads;  // (sequence, head) pairs that take long
  int nv = 4;
  while (nv > 1 && (nv > tiles || wide * ((tiles + nv - 1) / nv) < 512)) nv /= 2;
  const dim3 grid(p.heads, (tiles + nv - 1) / nv, p.num_seqs);
  if (nv == 4) hipLaunchKernelGGL((delta_scan_kernel<NT, 4>), grid, dim3(256), 0, s, p);
  else if (nv == 2) hipLaunchKernelGGL((delta_scan_kernel<NT, 2>), grid, dim3(256), 0, s, p);
  else hipLaunchKernelGGL((delta_scan_kernel<NT, 1>), grid, dim3(256), 0, s, p);
  LV_LAUNCH_CHECK();
  return 0;
}

template <typename T, int NT>
static int launch_chunks(const DeltaChunkParams& p, int rows, int max_query_len, hipStream_t s) {
  constexpr int smem = prepare_lds_floats(NT) * 4;
  if (smem > 64 * 1024)
    (void)hipFuncSetAttribute((const void*)delta_prepare_kernel<T, NT>, hipFuncAttributeMaxDynamicSharedMemorySize, smem);
  hipLaunchKernelGGL((delta_prepare_kernel<T, NT>), dim3(p.heads, rows / kChunk + p.num_seqs), dim3(256), smem, s, p);
  LV_LAUNCH_CHECK();
  return launch_scan<NT>(p, rows, max_query_len, s);
}

}  // namespace lvllm

using namespace lvllm;

static int check_sizes(const lvllm_delta_sizes& d) {
  LV_CHECK(d.dk > 0 && d.dk <= 256 && d.dv > 0 && d.dv <= 1024, "key size must be in 1 .. 256, value size in 1 .. 1024");
  LV_CHECK(d.kv_heads > 0 && d.heads % d.kv_heads == 0 && d.heads <= 65535, "heads share their keys evenly");
  return 0;
}

extern "C" int lvllm_delta_step(void* out, int64_t out_stride, const void* x, int64_t x_stride, const void* u, const void* z,
                                const void* beta, const float* conv_weight, int taps, int channels, float* conv_state,
                                int64_t conv_stride, const void* decay_w, int decay_rank, const void* gate_w, int gate_rank,
                                const float* decay_scale, const float* decay_bias, const float* norm_weight, float eps,
                                const lvllm_delta_sizes* sizes, float* state, int64_t state_stride, const int32_t* state_slots,
                                int num_slots, const int32_t* seq_lens, int num_seqs, int dtype, void* stream) {
  if (num_seqs == 0) return 0;
  const lvllm_delta_sizes& d = *sizes;
  if (int rc = check_sizes(d)) return rc;
  LV_CHECK(taps >= 1 && taps <= kMaxTaps && decay_rank > 0 && decay_rank <= 512 && gate_rank > 0 && gate_rank <= 512,
           "1 .. 16 taps, ranks of 1 .. 512");
  LV_CHECK(d.kv_heads * d.dk <= d.k_at && d.k_at + d.kv_heads * d.dk <= d.v_at && d.v_at + d.heads * d.dv <= channels,
           "q, k and v overlap");
  LV_CHECK(conv_stride >= (int64_t)taps * channels && state_stride >= (int64_t)d.heads * d.dk * d.dv &&
               ((d.dv & 3) != 0 || (state_stride & 3) == 0), "state slots overlap or are unaligned");
  LV_CHECK(num_seqs <= 65535 && (((uintptr_t)decay_w | (uintptr_t)gate_w) & 15) == 0, "too many sequences, or unaligned weights");
  DeltaStepParams p{};
  p.out = out; p.out_stride = out_stride; p.x = x; p.x_stride = x_stride; p.u = u; p.z = z; p.beta = beta;
  p.conv_weight = conv_weight; p.taps = taps; p.channels = channels; p.conv_state = conv_state; p.conv_stride = conv_stride;
  p.decay_w = decay_w; p.decay_rank = decay_rank; p.gate_w = gate_w; p.gate_rank = gate_rank; p.decay_scale = decay_scale;
  p.decay_bias = decay_bias; p.norm_weight = norm_weight; p.eps = eps; p.state = state; p.state_stride = state_stride;
  p.state_slots = state_slots; p.num_slots = num_slots; p.seq_lens = seq_lens; p.num_seqs = num_seqs; p.heads = d.heads;
  p.kv_heads = d.kv_heads; p.dk = d.dk; p.dv = d.dv; p.k_at = d.k_at; p.v_at = d.v_at; p.q_scale = d.q_scale;
  const bool vec = (d.dv & 3) == 0;
  const int rgs = 256 / step_columns(d.dv, vec ? 4 : 1), pre = vec && d.dv <= 1024 ? (d.dk + rgs - 1) / rgs : 1 << 20;
  const size_t smem = (size_t)StepLds(d.dk, d.dv, decay_rank, gate_rank, rgs).total * sizeof(float);
  const dim3 grid(d.heads, num_seqs);
  hipStream_t s = (hipStream_t)stream;
  LV_DISPATCH_F32_BF16(dtype, {
    if (pre <= 4) hipLaunchKernelGGL((delta_step_kernel<scalar_t, 4, 4>), grid, dim3(256), smem, s, p);
    else if (pre <= 8) hipLaunchKernelGGL((delta_step_kernel<scalar_t, 8, 4>), grid, dim3(256), smem, s, p);
    else if (pre <= 16) hipLaunchKernelGGL((delta_step_kernel<scalar_t, 16, 4>), grid, dim3(256), smem, s, p);
    else if (vec) hipLaunchKernelGGL((delta_step_kernel<scalar_t, 0, 4>), grid, dim3(256), smem, s, p);
    else hipLaunchKernelGGL((delta_step_kernel<scalar_t, 0, 1>), grid, dim3(256), smem, s, p);
  });
  LV_LAUNCH_CHECK();
  return 0;
}

extern "C" int64_t lvllm_delta_chunks_workspace_bytes(const lvllm_delta_sizes* sizes, int rows, int num_seqs) {
  const int64_t per_row = (int64_t)sizes->heads * (((sizes->dk + 3) & ~3) + sizes->dv);
  return ((int64_t)rows * per_row + 4 +
          ((int64_t)rows / kChunk + num_seqs) * sizes->heads * chunk_layout(sizes->dk, sizes->dv).size()) * 4;
}

extern "C" int lvllm_delta_chunks(void* out, int64_t out_stride, const void* y, int64_t y_stride, const void* u, const void* beta,
                                  int64_t u_stride, const float* a_t, int decay_rank, const float* decay_scale,
                                  const float* decay_bias, const void* gate, int64_t gate_stride, const float* norm_weight,
                                  float eps, const lvllm_delta_sizes* sizes, float* state, int64_t state_stride,
                                  const int32_t* state_slots, int num_slots, const int32_t* query_start_loc,
                                  const int32_t* seq_lens, int num_seqs, int rows, int max_query_len, void* workspace,
                                  int64_t workspace_bytes, int dtype, void* stream) {
  if (num_seqs == 0 || rows == 0) return 0;
  const lvllm_delta_sizes& d = *sizes;
  if (int rc = check_sizes(d)) return rc;
  LV_CHECK(num_seqs <= 65535 && rows / kChunk + num_seqs <= 65535 && max_query_len > 0, "too many sequences or rows");
  LV_CHECK(state_stride >= (int64_t)d.heads * d.dk * d.dv, "state slots overlap");
  LV_CHECK(workspace != nullptr && workspace_bytes >= lvllm_delta_chunks_workspace_bytes(sizes, rows, num_seqs),
           "workspace too small (see lvllm_delta_chunks_workspace_bytes)");
  LV_CHECK(dtype == LVLLM_BF16 || dtype == LVLLM_F32, "bfloat16 or float32");
  DeltaChunkParams p{};
  float* ws = (float*)workspace;
  p.layout = chunk_layout(d.dk, d.dv);
  p.chunks = ws;
  ws += ((int64_t)rows / kChunk + num_seqs) * d.heads * p.layout.size();
  float* log_decay = ws;
  ws += ((int64_t)rows * d.heads * d.dk + 3) & ~(int64_t)3;
  p.o = ws;
  p.log_decay = log_decay; p.y = y; p.y_stride = y_stride; p.beta = beta; p.beta_stride = u_stride; p.state = state;
  p.state_stride = state_stride; p.state_slots = state_slots; p.num_slots = num_slots; p.query_start_loc = query_start_loc;
  p.seq_lens = seq_lens; p.num_seqs = num_seqs; p.heads = d.heads; p.kv_heads = d.kv_heads; p.dk = d.dk; p.dv = d.dv;
  p.k_at = d.k_at; p.v_at = d.v_at; p.q_scale = d.q_scale;
  hipStream_t s = (hipStream_t)stream;
  if (int rc = launch_log_decay(log_decay, u, u_stride, a_t, decay_bias, kDecaySoftplus, 1.f, decay_scale, rows, decay_rank,
                                d.heads * d.dk, dtype, s)) return rc;
  int rc = 0;
  LV_DISPATCH_F32_BF16(dtype, {
    const int nt = key_tiles(d.dk);
    rc = nt == 1 ? launch_chunks<scalar_t, 1>(p, rows, max_query_len, s)
         : nt == 2 ? launch_chunks<scalar_t, 2>(p, rows, max_query_len, s) : launch_chunks<scalar_t, 4>(p, rows, max_query_len, s);
  });
  if (rc) return rc;
  return launch_head_norm_gate<false>(out, out_stride, p.o, gate, gate_stride, norm_weight, 0, eps, 1.f, rows, d.heads, d.dv,
                                      dtype, s);
}
