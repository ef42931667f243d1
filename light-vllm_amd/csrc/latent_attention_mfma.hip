// The absorbed body of latent_attention.h on bf16 MFMAs: scores and weighted sums on the cached rows themselves.
//
// A workgroup serves 16 CT (token, head) columns of one sequence and one share of the keys; the columns' window is walked in
// tiles of 64 keys = 4 pages.  Pages are contiguous in memory and go straight to LDS (two stages: the next tile's copies are
// in flight while one is used), the 16-byte chunks of a row exchanged so that row reads are free of bank conflicts.  Four
// waves work on 16 columns:
//   * S^T = rows x q'^T: wave w scores the tile's page w; the columns' maxima meet in LDS;
//   * the probabilities go through LDS (64 keys x 16 columns of bf16);
//   * O^T += rows^T x P: wave w sums a quarter of the latent's entries; rows^T is read with the transposing LDS read.
// One read of a row serves both products and all 16 CT columns.  A second launch adds the shares, takes the sums out of
// latent space (V_h) and applies the gate.
#include <float.h>

#include "latent_attention.h"

namespace lvllm {

typedef __bf16 m_bf16x8_t __attribute__((ext_vector_type(8)));
typedef short m_i16x4_t __attribute__((ext_vector_type(4)));
typedef float m_f32x4_t __attribute__((ext_vector_type(4)));
typedef unsigned int m_u32x4_t __attribute__((ext_vector_type(4)));
typedef unsigned int m_u32x2_t __attribute__((ext_vector_type(2)));

__device__ __forceinline__ m_f32x4_t mfma16(m_u32x4_t a, m_u32x4_t b, m_f32x4_t c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(m_bf16x8_t, a), __builtin_bit_cast(m_bf16x8_t, b), c, 0, 0,
                                                 0);
}

// What chunk numbers of row r of a page are exchanged by (an exclusive or): rows whose first bank is the same differ.
template <int NK>
__device__ __forceinline__ int exchange(int r) {
  return NK % 4 == 0 ? r & 15 : NK % 2 == 0 ? (r >> 1) & 7 : (r >> 2) & 3;
}

// everything written to LDS so far is seen by the workgroup; copies in flight stay in flight
__device__ __forceinline__ void lds_barrier() { asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory"); }

// NC, NR: latent and rotated part in units of 32 entries
template <int NC, int NR, int CT>
__global__ __launch_bounds__(256 * CT, 1) void latent_attention_mfma_kernel(const LatentAttnParams p) {
  constexpr int NK = NC + NR, RE = 32 * NK, CP = 32 * NC;
  constexpr int RC = 4 * NK, RB = 64 * NK;  // 16-byte chunks and bytes of a row
  constexpr int kStage = 64 * RB;
  constexpr int COPIES = (NK + CT - 1) / CT;  // of 1 KiB, per wave and tile: a page is NK KiB
  constexpr int NT = NC / 2;               // 16-entry tiles of O a wave owns
  constexpr int PP = 72;                   // elements between columns of P
  extern __shared__ __attribute__((aligned(16))) char tile[];  // [2][64][RB]
  __shared__ __attribute__((aligned(16))) uint16_t sp[CT][16 * PP];
  __shared__ float sm[CT][4][16];
  const int lane = threadIdx.x & 63;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int kg = CT == 1 ? wave : wave & 3, ct = CT == 1 ? 0 : wave >> 2;
  const int g = lane >> 4, c = lane & 15;
  const int seq = blockIdx.y, share = blockIdx.z;
  const int qbeg = p.query_start_loc[seq], qlen = p.query_start_loc[seq + 1] - qbeg;
  if (qlen <= 0 || qlen > p.absorbed_max) return;
  const int ncols = qlen * p.heads, col_wg = blockIdx.x * 16 * CT;
  if (col_wg >= ncols) return;
  const int ctx = p.seq_lens[seq] - qlen;
  const int col = col_wg + 16 * ct + c;
  const bool col_ok = col < ncols;
  const int tok = min(col, ncols - 1) / p.heads, head = min(col, ncols - 1) - tok * p.heads;
  const int64_t at = (int64_t)(qbeg + tok) * p.heads + head;
  const int pos = ctx + tok, low = first_key(pos, p.window);
  const int wg_first = ctx + col_wg / p.heads, wg_last = ctx + (min(col_wg + 16 * CT, ncols) - 1) / p.heads;
  const int lo = first_key(wg_first, p.window) & ~15;
  const int ntiles = wg_last >= 0 ? (wg_last + 1 - lo + 63) / 64 : 0;
  const int per = (ntiles + p.nsplit - 1) / p.nsplit;
  const int t0 = share * per, t1 = min(t0 + per, ntiles);

  const int32_t* table = p.block_tables + (int64_t)seq * p.max_blocks;
  int from[COPIES];  // elements from the page's start that this lane copies
#pragma unroll
  for (int j = 0; j < COPIES; ++j) {
    const int i = (j * CT + ct) * 64 + lane, r = i / RC;
    from[j] = r * RE + ((i - r * RC) ^ exchange<NK>(r)) * 8;
  }
  auto page_of = [&](int t) { return table[min(lo / 16 + 4 * t + kg, p.max_blocks - 1)]; };
  auto copy = [&](int t, int page) __attribute__((always_inline)) {
    const int64_t blk = min(max(page, 0), p.max_block);
    const uint16_t* src = (const uint16_t*)p.cache + blk * p.block_stride;
    char* dst = tile + ((t - t0) & 1) * kStage + kg * 16 * RB;
#pragma unroll
    for (int j = 0; j < COPIES; ++j)
      if (j * CT + ct < NK)
        __builtin_amdgcn_global_load_lds((const __attribute__((address_space(1))) void*)(src + from[j]),
                                         (__attribute__((address_space(3))) void*)(dst + (j * CT + ct) * 1024), 16, 0, 0);
  };
  if (t0 < t1) copy(t0, page_of(t0));
  int page = page_of(t0 + 1);  // (looked up a tile ahead)
  m_u32x4_t qf[NK];
  {
    const uint16_t* q = (const uint16_t*)p.q + at * RE + 8 * g;
#pragma unroll
    for (int j = 0; j < NK; ++j) qf[j] = *reinterpret_cast<const m_u32x4_t*>(q + 32 * j);
  }
  __builtin_amdgcn_s_waitcnt(0 | (7 << 4) | (15 << 8));  // (q has landed: nothing in the loop waits for it)
  const float sl = p.scale * 1.4426950408889634f;
  float m = -1e30f, l = 0.f;
  m_f32x4_t o[NT];
#pragma unroll
  for (int i = 0; i < NT; ++i) o[i] = m_f32x4_t{0.f, 0.f, 0.f, 0.f};
  const int kx = exchange<NK>(c), krow = (kg * 16 + c) * RB;
  const int vr = 8 * g + (c >> 2), vx0 = exchange<NK>(vr & 15), vx1 = exchange<NK>((vr + 4) & 15);
  const int vc = kg * NT * 2 + ((c & 3) >> 1), vb = (c & 1) * 8;
  typedef __attribute__((address_space(3))) m_i16x4_t* lds_tr_t;

  for (int t = t0; t < t1; ++t) {
    // the copies of this tile have landed, for every wave; everyone is done with the tile before
    __builtin_amdgcn_s_waitcnt(0 | (7 << 4) | (15 << 8));
    asm volatile("s_barrier" ::: "memory");
    if (t + 1 < t1) copy(t + 1, page);
    page = page_of(t + 2);
    const char* st = tile + ((t - t0) & 1) * kStage;
    m_f32x4_t s{0.f, 0.f, 0.f, 0.f}, s2{0.f, 0.f, 0.f, 0.f};
    constexpr int W = NK < 6 ? NK : 6;  // fragments read ahead
    m_u32x4_t k[W];
    auto kread = [&](int j) { return *reinterpret_cast<const m_u32x4_t*>(st + krow + (((4 * j + g) ^ kx) * 16)); };
#pragma unroll
    for (int j = 0; j < W; ++j) k[j] = kread(j);
    __builtin_amdgcn_sched_barrier(0);
#pragma unroll
    for (int j = 0; j < NK; ++j) {
      if (j & 1) s2 = mfma16(k[j % W], qf[j], s2);
      else s = mfma16(k[j % W], qf[j], s);
      if (j + W < NK) k[j % W] = kread(j + W);
      __builtin_amdgcn_sched_barrier(0);
    }
    s += s2;
    const int key0 = lo + 64 * t + 16 * kg + 4 * g;
#pragma unroll
    for (int r = 0; r < 4; ++r) s[r] = key0 + r <= pos && key0 + r >= low ? s[r] * sl : -FLT_MAX;
    float mx = fmaxf(fmaxf(s[0], s[1]), fmaxf(s[2], s[3]));
    mx = fmaxf(mx, __shfl_xor(mx, 16));
    mx = fmaxf(mx, __shfl_xor(mx, 32));
    if (g == 0) sm[ct][kg][c] = mx;
    lds_barrier();
    mx = fmaxf(fmaxf(sm[ct][0][c], sm[ct][1][c]), fmaxf(sm[ct][2][c], sm[ct][3][c]));
    if (__any(mx > m)) {
      const float mn = fmaxf(m, mx), corr = exp2f(m - mn);
      m = mn;
      l *= corr;
#pragma unroll
      for (int i = 0; i < NT; ++i) o[i] *= corr;
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) s[r] = __builtin_amdgcn_exp2f(s[r] - m);
    l += (s[0] + s[1]) + (s[2] + s[3]);
    {
      uint2 w;
      w.x = (uint32_t)BF16::from_float(s[0]) | ((uint32_t)BF16::from_float(s[1]) << 16);
      w.y = (uint32_t)BF16::from_float(s[2]) | ((uint32_t)BF16::from_float(s[3]) << 16);
      *reinterpret_cast<uint2*>(&sp[ct][c * PP + 16 * kg + 4 * g]) = w;
    }
    lds_barrier();
#pragma unroll
    for (int ks = 0; ks < 2; ++ks) {
      const m_u32x4_t pf = *reinterpret_cast<const m_u32x4_t*>(&sp[ct][c * PP + 32 * ks + 8 * g]);
      const char* v = st + (32 * ks + vr) * RB + vb;
      m_i16x4_t a[NT], b[NT];
#pragma unroll
      for (int i = 0; i < NT; ++i) {
        a[i] = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_tr_t)(v + (((vc + 2 * i) ^ vx0) * 16)));
        b[i] = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_tr_t)(v + 4 * RB + (((vc + 2 * i) ^ vx1) * 16)));
      }
      __builtin_amdgcn_sched_barrier(0);
#pragma unroll
      for (int i = 0; i < NT; ++i) {
        const m_u32x2_t ua = __builtin_bit_cast(m_u32x2_t, a[i]), ub = __builtin_bit_cast(m_u32x2_t, b[i]);
        o[i] = mfma16(m_u32x4_t{ua.x, ua.y, ub.x, ub.y}, pf, o[i]);
      }
    }
  }
  l += __shfl_xor(l, 16);
  l += __shfl_xor(l, 32);
  __syncthreads();
  if (g == 0) sm[ct][kg][c] = l;
  __syncthreads();
  if (!col_ok) return;
  const int64_t part = at * p.nsplit + share;
  float* out = p.part_o + part * CP + kg * NT * 16 + 4 * g;
#pragma unroll
  for (int i = 0; i < NT; ++i) *reinterpret_cast<m_f32x4_t*>(out + 16 * i) = o[i];
  if (kg == 0 && g == 0) {
    p.part_ml[2 * part] = m;
    p.part_ml[2 * part + 1] = (sm[ct][0][c] + sm[ct][1][c]) + (sm[ct][2][c] + sm[ct][3][c]);
  }
}

// The shares of R rows of one head -> their weighted sum o in latent space (bf16, as W's product reads it) -> out = V_h o * gate.
// grid (heads, rows / R); 8 waves add the shares of R rows' halves, then take every eighth 16-row tile of V_h.
template <int R>
__global__ __launch_bounds__(512) void latent_value_kernel(const LatentAttnParams p) {
  extern __shared__ __attribute__((aligned(16))) uint16_t so[];  // [R][cpad + 8]
  const int lane = threadIdx.x & 63;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int g = lane >> 4, c = lane & 15;
  const int head = blockIdx.x, row0 = blockIdx.y * R, ld = p.cpad + 8;
  constexpr int B = 16, S = 8;  // k-steps and shares in flight
  const int steps = p.cpad >> 5;
  const uint16_t* uv = (const uint16_t*)p.uv + ((int64_t)head * p.vpad + c) * p.cpad + 8 * g;
  m_u32x4_t w[B];
  auto fetch = [&](int n, int k0) __attribute__((always_inline)) {
#pragma unroll
    for (int j = 0; j < B; ++j)
      if (k0 + j < steps) w[j] = *reinterpret_cast<const m_u32x4_t*>(uv + (int64_t)n * 16 * p.cpad + 32 * (k0 + j));
  };
  // steps of single tokens: row i is sequence i; else the row's sequence tells whether it is in latent space at all
  const bool single = p.max_query_len == 1 && p.rows == p.num_seqs;
  auto absorbed = [&](int row) {
    if (single) return true;
    const int seq = find_seq(p.query_start_loc, p.num_seqs, row);
    return seq < p.num_seqs && p.query_start_loc[seq + 1] - p.query_start_loc[seq] <= p.absorbed_max;
  };
  if (wave * 16 < p.vpad) fetch(wave, 0);
  const int half = (p.cpad >> 1) >= 256 ? 2 : 1, part = p.cpad / half;  // (a lane takes 4 entries a turn)
  for (int i = wave; i < R * half; i += 8) {
    const int r = i / half, row = row0 + r, d0 = (i - r * half) * part;
    if (row >= p.rows || !absorbed(row)) {
      for (int d = d0 + lane; d < d0 + part; d += 64) so[r * ld + d] = 0;
      continue;
    }
    const int64_t at = ((int64_t)row * p.heads + head) * p.nsplit;
    const float ms = lane < p.nsplit ? p.part_ml[2 * (at + lane)] : -1e30f;
    const float ls = lane < p.nsplit ? p.part_ml[2 * (at + lane) + 1] : 0.f;
    float4 t[S];
    auto load = [&](int d, int s0) __attribute__((always_inline)) {
#pragma unroll
      for (int s = 0; s < S; ++s)
        if (s0 + s < p.nsplit) t[s] = *reinterpret_cast<const float4*>(p.part_o + (at + s0 + s) * p.cpad + d);
    };
    int d = d0 + lane * 4;
    if (d < d0 + part) load(d, 0);
    const float sink = p.sink != nullptr ? p.sink[head] * 1.4426950408889634f : -1e30f;
    const float m = fmaxf(wave_max(ms), sink);
    const float e = exp2f(ms - m);
    float l = wave_sum(ls * e);
    if (p.sink != nullptr) l += exp2f(sink - m);
    const float ws = l > 0.f ? e / l : 0.f;
    for (; d < d0 + part; d += 256) {
      float v[4] = {0.f, 0.f, 0.f, 0.f};
      for (int s0 = 0; s0 < p.nsplit; s0 += S) {
        if (s0 > 0 || d >= d0 + 256) load(d, s0);
#pragma unroll
        for (int s = 0; s < S; ++s)
          if (s0 + s < p.nsplit) {
            const float f = __builtin_bit_cast(float, __builtin_amdgcn_readlane(__builtin_bit_cast(int, ws), s0 + s));
            v[0] = fmaf(t[s].x, f, v[0]); v[1] = fmaf(t[s].y, f, v[1]); v[2] = fmaf(t[s].z, f, v[2]); v[3] = fmaf(t[s].w, f, v[3]);
          }
      }
      store4<BF16>(so + r * ld + d, v);
    }
  }
  const int row = row0 + c;
  bool mine = c < R && row < p.rows;
  float f = 1.f;
  if (mine && p.gate != nullptr)
    f = 1.f / (1.f + expf(-BF16::to_float(((const uint16_t*)p.gate)[row * p.gate_stride + head])));
  if (mine && !single) {
    const int seq = find_seq(p.query_start_loc, p.num_seqs, row);  // (padding rows get zeros)
    mine = seq >= p.num_seqs || p.query_start_loc[seq + 1] - p.query_start_loc[seq] <= p.absorbed_max;
  }
  __syncthreads();
  for (int n = wave; n * 16 < p.vpad; n += 8) {
    m_f32x4_t acc{0.f, 0.f, 0.f, 0.f};
    for (int k0 = 0; k0 < steps; k0 += B) {
      if (n != wave || k0 > 0) fetch(n, k0);
#pragma unroll
      for (int j = 0; j < B; ++j)
        if (k0 + j < steps) {
          m_u32x4_t x{0, 0, 0, 0};
          if (c < R) x = *reinterpret_cast<const m_u32x4_t*>(so + c * ld + 32 * (k0 + j) + 8 * g);
          acc = mfma16(w[j], x, acc);
        }
    }
    if (!mine) continue;
    uint16_t* out = (uint16_t*)p.out + row * p.out_stride + (int64_t)head * p.vdim + 16 * n + 4 * g;
#pragma unroll
    for (int r = 0; r < 4; ++r)
      if (16 * n + 4 * g + r < p.vdim) out[r] = BF16::from_float(acc[r] * f);
  }
}

template <int NC, int NR, int CT>
static void go(const LatentAttnParams& p, hipStream_t s) {
  constexpr int smem = 2 * 64 * 64 * (NC + NR);
  if (smem > 64 * 1024)
    (void)hipFuncSetAttribute((const void*)latent_attention_mfma_kernel<NC, NR, CT>,
                              hipFuncAttributeMaxDynamicSharedMemorySize, smem);
  const int64_t cols = (int64_t)p.heads * p.max_query_len;
  hipLaunchKernelGGL((latent_attention_mfma_kernel<NC, NR, CT>),
                     dim3((unsigned)((cols + 16 * CT - 1) / (16 * CT)), p.num_seqs, p.nsplit), dim3(256 * CT), smem, s, p);
}

bool latent_takes_mfma(int cpad, int rpad, int block_size, int dtype) {
  return dtype == LVLLM_BF16 && block_size == 16 && (cpad == 64 || cpad == 128 || cpad == 256 || cpad == 512) &&
         (rpad == 32 || rpad == 64);
}

template <int NC, int NR>
static void go_cols(const LatentAttnParams& p, hipStream_t s) {
  if ((int64_t)p.heads * p.max_query_len <= 16) go<NC, NR, 1>(p, s);
  else go<NC, NR, 2>(p, s);
}

int launch_latent_mfma(const LatentAttnParams& p, hipStream_t s) {
#define LV_LATENT_R(NC_)                    \
  if (p.rpad == 32) go_cols<NC_, 1>(p, s);  \
  else go_cols<NC_, 2>(p, s);               \
  break;
  switch (p.cpad) {
    case 64: LV_LATENT_R(2)
    case 128: LV_LATENT_R(4)
    case 256: LV_LATENT_R(8)
    case 512: LV_LATENT_R(16)
    default: LV_CHECK(false, "latent size");
  }
#undef LV_LATENT_R
  LV_LAUNCH_CHECK();
  LV_CHECK((p.rows + 3) / 4 <= 65535, "too many rows");
  if (p.rows <= 256)
    hipLaunchKernelGGL((latent_value_kernel<4>), dim3(p.heads, (p.rows + 3) / 4), dim3(512), 4 * (p.cpad + 8) * 2, s, p);
  else
    hipLaunchKernelGGL((latent_value_kernel<16>), dim3(p.heads, (p.rows + 15) / 16), dim3(512), 16 * (p.cpad + 8) * 2, s, p);
  LV_LAUNCH_CHECK();
  return 0;
}

}  // namespace lvllm
