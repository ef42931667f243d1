// The absorbed body of latent_attention.h on bf16 MFMAs: scores and weighted sums on the cached rows themselves.
//
// A workgroup serves 16 CT (token, head) columns of one sequence and one share of the keys; the columns' window is walked in
// tiles of 64 keys = 4 pages.  Pages are contiguous in memory and go to LDS row by row (16 bytes of padding between rows: row
// reads and transposed reads are free of bank conflicts), the next tile's loads in flight in registers meanwhile.  Four
// waves work on 16 columns:
//   * S^T = rows x q'^T: wave w scores the tile's page w; the columns' maxima meet in LDS;
//   * the probabilities go through LDS (64 keys x 16 columns of bf16);
//   * O^T += rows^T x P: wave w sums a quarter of the latent's entries; rows^T is read with the transposing LDS read.
// One read of a row serves both products and all 16 CT columns.  Shares meet in a second small launch.
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

// NC, NR: latent and rotated part in units of 32 entries
template <int NC, int NR, int CT>
__global__ __launch_bounds__(256 * CT, CT == 1 ? 2 : 1) void latent_attention_mfma_kernel(const LatentAttnParams p) {
  constexpr int NK = NC + NR, RE = 32 * NK, CP = 32 * NC;
  constexpr int RC = 4 * NK;               // 16-byte chunks of a row
  constexpr int PITCH = RE * 2 + 16;       // bytes between rows in LDS
  constexpr int LOADS = CT == 1 ? NK : (NK + 1) / 2;  // of 64 chunks, per wave: a page is 64 NK chunks
  constexpr int NT = NC / 2;               // 16-entry tiles of O a wave owns
  constexpr int PP = 72;                   // elements between columns of P
  extern __shared__ __attribute__((aligned(16))) char tile[];  // [64][PITCH]
  __shared__ __attribute__((aligned(16))) uint16_t sp[CT][16 * PP];
  __shared__ float sm[CT][4][16];
  const int lane = threadIdx.x & 63;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int kg = wave & 3, ct = wave >> 2;
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

  m_u32x4_t qf[NK];
  {
    const uint16_t* q = (const uint16_t*)p.q + at * RE + 8 * g;
#pragma unroll
    for (int j = 0; j < NK; ++j) qf[j] = *reinterpret_cast<const m_u32x4_t*>(q + 32 * j);
  }
  const int32_t* table = p.block_tables + (int64_t)seq * p.max_blocks;
  m_u32x4_t st[LOADS];
  auto fetch = [&](int t) __attribute__((always_inline)) {
    const int64_t blk = min(max(table[min(lo / 16 + 4 * t + kg, p.max_blocks - 1)], 0), p.max_block);
    const uint16_t* src = (const uint16_t*)p.cache + blk * p.block_stride;
#pragma unroll
    for (int j = 0; j < LOADS; ++j) {
      const int i = (ct * LOADS + j) * 64 + lane;
      if (CT == 1 || ct * LOADS + j < NK) st[j] = *reinterpret_cast<const m_u32x4_t*>(src + i * 8);
    }
  };
  auto put = [&]() __attribute__((always_inline)) {
#pragma unroll
    for (int j = 0; j < LOADS; ++j) {
      const int i = (ct * LOADS + j) * 64 + lane;
      if (CT == 1 || ct * LOADS + j < NK)
        *reinterpret_cast<m_u32x4_t*>(tile + (kg * 16 + i / RC) * PITCH + (i % RC) * 16) = st[j];
    }
  };
  const float sl = p.scale * 1.4426950408889634f;
  float m = -1e30f, l = 0.f;
  m_f32x4_t o[NT];
#pragma unroll
  for (int i = 0; i < NT; ++i) o[i] = m_f32x4_t{0.f, 0.f, 0.f, 0.f};
  const char* krow = tile + (kg * 16 + c) * PITCH + 16 * g;
  const char* vrow = tile + (8 * g + (c >> 2)) * PITCH + (kg * NT * 16 + 4 * (c & 3)) * 2;
  typedef __attribute__((address_space(3))) m_i16x4_t* lds_tr_t;

  if (t0 < t1) fetch(t0);
  for (int t = t0; t < t1; ++t) {
    put();
    __syncthreads();
    if (t + 1 < t1) fetch(t + 1);
    m_f32x4_t s{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int j = 0; j < NK; ++j) s = mfma16(*reinterpret_cast<const m_u32x4_t*>(krow + 64 * j), qf[j], s);
    const int key0 = lo + 64 * t + 16 * kg + 4 * g;
#pragma unroll
    for (int r = 0; r < 4; ++r) s[r] = key0 + r <= pos && key0 + r >= low ? s[r] * sl : -FLT_MAX;
    float mx = fmaxf(fmaxf(s[0], s[1]), fmaxf(s[2], s[3]));
    mx = fmaxf(mx, __shfl_xor(mx, 16));
    mx = fmaxf(mx, __shfl_xor(mx, 32));
    if (g == 0) sm[ct][kg][c] = mx;
    __syncthreads();
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
    __syncthreads();
#pragma unroll
    for (int ks = 0; ks < 2; ++ks) {
      const m_u32x4_t pf = *reinterpret_cast<const m_u32x4_t*>(&sp[ct][c * PP + 32 * ks + 8 * g]);
#pragma unroll
      for (int i = 0; i < NT; ++i) {
        const char* v = vrow + 32 * ks * PITCH + 32 * i;
        const m_i16x4_t a = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_tr_t)v);
        const m_i16x4_t b = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_tr_t)(v + 4 * PITCH));
        const m_u32x2_t ua = __builtin_bit_cast(m_u32x2_t, a), ub = __builtin_bit_cast(m_u32x2_t, b);
        o[i] = mfma16(m_u32x4_t{ua.x, ua.y, ub.x, ub.y}, pf, o[i]);
      }
    }
    __syncthreads();
  }
  l += __shfl_xor(l, 16);
  l += __shfl_xor(l, 32);
  if (g == 0) sm[ct][kg][c] = l;
  __syncthreads();
  l = (sm[ct][0][c] + sm[ct][1][c]) + (sm[ct][2][c] + sm[ct][3][c]);
  if (!col_ok) return;
  if (p.nsplit > 1) {
    const int64_t part = at * p.nsplit + share;
    float* out = p.part_o + part * CP + kg * NT * 16 + 4 * g;
#pragma unroll
    for (int i = 0; i < NT; ++i) *reinterpret_cast<m_f32x4_t*>(out + 16 * i) = o[i];
    if (kg == 0 && g == 0) {
      p.part_ml[2 * part] = m;
      p.part_ml[2 * part + 1] = l;
    }
  } else {
    const float f = l > 0.f ? 1.f / l : 0.f;
    uint16_t* out = (uint16_t*)p.out + at * CP + kg * NT * 16 + 4 * g;
#pragma unroll
    for (int i = 0; i < NT; ++i) {
      const float v[4] = {o[i][0] * f, o[i][1] * f, o[i][2] * f, o[i][3] * f};
      store4<BF16>(out + 16 * i, v);
    }
  }
}

// Shares of one (row, head) -> out
__global__ __launch_bounds__(128) void latent_reduce_kernel(const LatentAttnParams p) {
  const int row = blockIdx.x, head = blockIdx.y;
  const int seq = find_seq(p.query_start_loc, p.num_seqs, row);
  if (seq >= p.num_seqs) return;
  if (p.query_start_loc[seq + 1] - p.query_start_loc[seq] > p.absorbed_max) return;
  const int64_t at = ((int64_t)row * p.heads + head) * p.nsplit;
  float m = -1e30f;
  for (int s = 0; s < p.nsplit; ++s) m = fmaxf(m, p.part_ml[2 * (at + s)]);
  float l = 0.f;
  for (int s = 0; s < p.nsplit; ++s) l += p.part_ml[2 * (at + s) + 1] * exp2f(p.part_ml[2 * (at + s)] - m);
  const float f = l > 0.f ? 1.f / l : 0.f;
  for (int d = threadIdx.x * 4; d < p.cpad; d += 512) {
    float v[4] = {0.f, 0.f, 0.f, 0.f};
    for (int s = 0; s < p.nsplit; ++s) {
      const float w = exp2f(p.part_ml[2 * (at + s)] - m) * f;
      const float4 t = *reinterpret_cast<const float4*>(p.part_o + (at + s) * p.cpad + d);
      v[0] = fmaf(t.x, w, v[0]); v[1] = fmaf(t.y, w, v[1]); v[2] = fmaf(t.z, w, v[2]); v[3] = fmaf(t.w, w, v[3]);
    }
    store4<BF16>((uint16_t*)p.out + ((int64_t)row * p.heads + head) * p.cpad + d, v);
  }
}

template <int NC, int NR, int CT>
static void go(const LatentAttnParams& p, hipStream_t s) {
  constexpr int smem = 64 * (64 * (NC + NR) + 16);
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
  if (p.nsplit > 1) {
    hipLaunchKernelGGL(latent_reduce_kernel, dim3(p.rows, p.heads), dim3(128), 0, s, p);
    LV_LAUNCH_CHECK();
  }
  return 0;
}

}  // namespace lvllm
