// The chunk body of head_attention.h: causal attention of prompt portions over the paged cache on 32x32x16 bf16 MFMAs.
//
// A workgroup is 4 waves = 128 columns, a column being a (query token, head of the GQA group, map) triple; the waves share one
// stream of 64-key tiles through LDS (two stages, one barrier per tile, the next tile's global loads in flight meanwhile).
// With two maps, waves 0 and 1 take the first one, waves 2 and 3 the second one of the same 64 (token, head) pairs: each reads
// its half of the keys, and the two results meet in LDS at the end.
//   * S^T = K Q^T: a lane holds 32 keys of ONE column, so the column's maximum is in-lane plus one exchange of halves;
//   * the cache layouts are the operand layouts: a K fragment is a 16-byte chunk per lane of [kpad / 8][16][8], a V^T
//     fragment 8 consecutive tokens of a [vpad][16] row.  K goes to LDS verbatim; V's chunks are permuted on the way so
//     that a fragment read is 32 consecutive chunks;
//   * probabilities never move between lanes: MFMA row i of S^T holds a permuted key (groups of four 1 and 2 of every 16
//     trade places), which makes a lane's accumulators the consecutive keys that P V wants as its B operand;
//   * accumulators are rescaled only when a column's maximum grew;
//   * tiles of kept first keys come ahead of the window's.
#pragma once
#include <float.h>

#include "head_attention.h"

namespace lvllm {

__device__ __forceinline__ h_f32x16_t mfma32(h_u32x4_t a, h_u32x4_t b, h_f32x16_t c) {
  return __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(h_bf16x8_t, a), __builtin_bit_cast(h_bf16x8_t, b), c,
                                                 0, 0, 0);
}

template <int NK, int NV, int MAPS>
__global__ __launch_bounds__(256, NK + NV <= 10 ? 2 : 1) void head_prefill_kernel(const HeadAttnParams p) {
  constexpr int KP = 32 * NK, VP = 32 * NV, KS = 2 * NK / MAPS;  // KS: k-steps of a column
  constexpr int kPrefillCols = 128 / MAPS;                       // (token, head) pairs of a workgroup
  constexpr int kKBlock = KP * 16 * 2, kVBlock = VP * 16 * 2;  // bytes of a block's head slice
  constexpr int kImageK = 4 * kKBlock, kStage = kImageK + 4 * kVBlock;
  extern __shared__ __attribute__((aligned(16))) char smem[];
  const int lane = threadIdx.x & 63;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int lc = lane & 31, hi = lane >> 5;
  const int map = MAPS == 2 ? wave >> 1 : 0, cwave = MAPS == 2 ? wave & 1 : wave;
  const int kvh = blockIdx.x, seq = blockIdx.z;
  const int tile_q = gridDim.y - 1 - blockIdx.y;  // the end of the chunk, which sees the most keys, first
  const int G = p.heads / p.kv_heads;
  const int qbeg = p.query_start_loc[seq], qlen = p.query_start_loc[seq + 1] - qbeg;
  const int ncols = qlen * G;
  if (qlen <= 0 || qlen < p.min_query_len || takes_decode_body(qlen, G * MAPS) || tile_q * kPrefillCols >= ncols) return;
  const int ctx = p.seq_lens[seq] - qlen;
  if (ctx < 0) return;
  const int col0 = tile_q * kPrefillCols + cwave * 32;
  const int col = min(col0 + lc, ncols - 1);
  const bool col_ok = col0 + lc < ncols;
  const int tok = col / G, head = kvh * G + (col - tok * G);
  const int64_t row = qbeg + tok;
  const int pos = ctx + tok, low = first_seen(p, pos);  // the last and the first key this lane's column sees
  const int wg_last = ctx + (min(tile_q * kPrefillCols + kPrefillCols, ncols) - 1) / G;
  const bool wave_ok = col0 < ncols;
  const int wave_first = ctx + min(col0, ncols - 1) / G, wave_last = ctx + min(col0 + 31, ncols - 1) / G;
  const int wave_low = first_seen(p, wave_first), wave_all = first_seen(p, wave_last);
  const int tile0 = first_seen(p, ctx + tile_q * kPrefillCols / G) / 64;
  const int kept = min((p.keep_first + 63) / 64, tile0);  // tiles of kept keys ahead of the window's
  const int ntiles = wg_last / 64 + 1 - tile0 + kept;
  auto tile_of = [&](int t) { return t < kept ? t : t - kept + tile0; };

  h_u32x4_t qf[KS];
  {
    const uint16_t* q = (const uint16_t*)p.q + (row * p.heads + head) * KP + map * (KP / MAPS) + 8 * hi;
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) qf[ks] = *reinterpret_cast<const h_u32x4_t*>(q + 16 * ks);
  }
  const int32_t* table = p.block_tables + (int64_t)seq * p.max_blocks;
  const uint16_t* kc = (const uint16_t*)p.k_cache + (int64_t)kvh * KP * 16;
  const uint16_t* vc = (const uint16_t*)p.v_cache + (int64_t)kvh * VP * 16;
  h_u32x4_t kreg[NK], vreg[NV];
  auto fetch = [&](int tile) __attribute__((always_inline)) {
    int64_t blk[4];
#pragma unroll
    for (int b = 0; b < 4; ++b) blk[b] = min(max(table[min(tile * 4 + b, p.max_blocks - 1)], 0), p.max_block);
#pragma unroll
    for (int j = 0; j < NK; ++j) {
      const int b = (wave + 4 * j) / NK, w = (wave + 4 * j) - b * NK;  // 64-chunk group w of block b
      const int64_t bk = b == 0 ? blk[0] : b == 1 ? blk[1] : b == 2 ? blk[2] : blk[3];
      kreg[j] = *reinterpret_cast<const h_u32x4_t*>(kc + bk * p.k_block_stride + (w * 64 + lane) * 8);
    }
#pragma unroll
    for (int j = 0; j < NV; ++j) {
      const int b = (wave + 4 * j) / NV, w = (wave + 4 * j) - b * NV;
      const int64_t bk = b == 0 ? blk[0] : b == 1 ? blk[1] : b == 2 ? blk[2] : blk[3];
      vreg[j] = *reinterpret_cast<const h_u32x4_t*>(vc + bk * p.v_block_stride + (w * 64 + lane) * 8);
    }
  };
  auto put = [&](int stage) __attribute__((always_inline)) {
    char* base = smem + stage * kStage;
#pragma unroll
    for (int j = 0; j < NK; ++j) {
      const int b = (wave + 4 * j) / NK, w = (wave + 4 * j) - b * NK;
      *reinterpret_cast<h_u32x4_t*>(base + b * kKBlock + (w * 64 + lane) * 16) = kreg[j];
    }
#pragma unroll
    for (int j = 0; j < NV; ++j) {  // chunk `lane` of a 32-row group: row lane >> 1, tokens 8 * (lane & 1) ..
      const int b = (wave + 4 * j) / NV, w = (wave + 4 * j) - b * NV;
      *reinterpret_cast<h_u32x4_t*>(base + kImageK + b * kVBlock + (w * 64 + (lane & 1) * 32 + (lane >> 1)) * 16) = vreg[j];
    }
  };

  const ScoreScale score(p);
  float m = -1e30f, l = 0.f;
  h_f32x16_t o[NV];
#pragma unroll
  for (int i = 0; i < NV; ++i) o[i] = h_f32x16_t{};
  // MFMA row lc of S^T is key perm(lc) of the 32: groups of four 1 and 2 of every 16 trade places
  const int r16 = lc & 15, grp = r16 >> 2;
  const int key16 = (((grp & 1) << 1 | grp >> 1) << 2) | (r16 & 3);
  const int klds = (lc >> 4) * kKBlock + map * (kKBlock / MAPS) + (hi * 16 + key16) * 16;
  const int vlds = kImageK + lane * 16;  // (hi * 32 + lc) * 16

  fetch(tile_of(0));
  put(0);
  __syncthreads();
  for (int t = 0; t < ntiles; ++t) {
    const bool more = t + 1 < ntiles;
    if (more) fetch(tile_of(t + 1));
    const int k0 = tile_of(t) * 64;
    if (wave_ok && k0 <= wave_last && (k0 + 63 >= wave_low || k0 < p.keep_first)) {
      const char* base = smem + (t & 1) * kStage;
      h_f32x16_t s[2] = {h_f32x16_t{}, h_f32x16_t{}};
#pragma unroll
      for (int ks = 0; ks < KS; ++ks) {
        const h_u32x4_t a0 = *reinterpret_cast<const h_u32x4_t*>(base + klds + ks * 512);
        const h_u32x4_t a1 = *reinterpret_cast<const h_u32x4_t*>(base + klds + 2 * kKBlock + ks * 512);
        s[0] = mfma32(a0, qf[ks], s[0]);
        s[1] = mfma32(a1, qf[ks], s[1]);
      }
      if (score.cap > 0.f) {
#pragma unroll
        for (int h = 0; h < 2; ++h)
#pragma unroll
          for (int i = 0; i < 16; ++i) s[h][i] = score.capped(s[h][i]);
      } else {
#pragma unroll
        for (int h = 0; h < 2; ++h)
#pragma unroll
          for (int i = 0; i < 16; ++i) s[h][i] *= score.mul;
      }
      if (k0 + 63 > wave_first || k0 < wave_all) {  // the diagonal or the window's edge passes through it for some column
#pragma unroll
        for (int h = 0; h < 2; ++h)
#pragma unroll
          for (int i = 0; i < 16; ++i) {
            const int key = k0 + 32 * h + 16 * (i >> 3) + 8 * hi + (i & 7);
            s[h][i] = sees(p, key, pos, low) ? s[h][i] : -FLT_MAX;
          }
      }
      float mx = fmaxf(s[0][0], s[1][0]);
#pragma unroll
      for (int i = 1; i < 16; ++i) mx = fmaxf(mx, fmaxf(s[0][i], s[1][i]));
      mx = fmaxf(mx, __shfl_xor(mx, 32));
      if (__any(mx > m)) {
        const float mn = fmaxf(m, mx), corr = exp2f(m - mn);
        m = mn;
        l *= corr;
#pragma unroll
        for (int i = 0; i < NV; ++i) o[i] *= corr;
      }
      float sum = 0.f;
#pragma unroll
      for (int h = 0; h < 2; ++h)
#pragma unroll
        for (int i = 0; i < 16; ++i) {
          s[h][i] = __builtin_amdgcn_exp2f(s[h][i] - m);
          sum += s[h][i];
        }
      l += sum;
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        h_u32x4_t pf;
#pragma unroll
        for (int r = 0; r < 4; ++r) pf[r] = pack_bf16(s[j >> 1][8 * (j & 1) + 2 * r], s[j >> 1][8 * (j & 1) + 2 * r + 1]);
#pragma unroll
        for (int i = 0; i < NV; ++i) {
          const h_u32x4_t vf = *reinterpret_cast<const h_u32x4_t*>(base + vlds + j * kVBlock + i * 1024);
          o[i] = mfma32(vf, pf, o[i]);
        }
      }
    }
    if (more) put((t + 1) & 1);
    __syncthreads();
  }
  l += __shfl_xor(l, 32);
  l += sink_term(p, head, m);
  float f = 1.f / l;
  if constexpr (MAPS == 2) {
    constexpr int LD = VP + 4;
    float* other = reinterpret_cast<float*>(smem) + (cwave * 32 + lc) * LD + 4 * hi;  // the second map's result
    if (map == 1) {
#pragma unroll
      for (int i = 0; i < NV; ++i)
#pragma unroll
        for (int r4 = 0; r4 < 4; ++r4)
          *reinterpret_cast<float4*>(other + 32 * i + 8 * r4) =
              float4{o[i][4 * r4] * f, o[i][4 * r4 + 1] * f, o[i][4 * r4 + 2] * f, o[i][4 * r4 + 3] * f};
    }
    __syncthreads();
    if (map == 1) return;
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < NV; ++i)
#pragma unroll
      for (int r4 = 0; r4 < 4; ++r4) {
        const float4 b = *reinterpret_cast<const float4*>(other + 32 * i + 8 * r4);
        const float bv[4] = {b.x, b.y, b.z, b.w};
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const float v = fmaf(-p.map_weight, bv[r], o[i][4 * r4 + r] * f);
          o[i][4 * r4 + r] = v;
          ss = fmaf(v, v, ss);
        }
      }
    ss += __shfl_xor(ss, 32);
    f = 1.f / sqrtf(ss / (float)p.vdim + p.map_eps);
  }
  if (!col_ok) return;
  f *= gate_of<BF16>(p, row, head);
  uint16_t* out = (uint16_t*)p.out + row * p.out_stride + (int64_t)head * p.vdim;
  const bool vec = ((p.vdim | (int)p.out_stride) & 3) == 0 && (((uintptr_t)p.out) & 7) == 0;
#pragma unroll
  for (int i = 0; i < NV; ++i)
#pragma unroll
    for (int r4 = 0; r4 < 4; ++r4) {
      const int d = 32 * i + 8 * r4 + 4 * hi;
      if (vec) {
        if (d < p.vdim) {
          const float v[4] = {o[i][4 * r4] * f, o[i][4 * r4 + 1] * f, o[i][4 * r4 + 2] * f, o[i][4 * r4 + 3] * f};
          store4<BF16>(out + d, v);
        }
      } else {
#pragma unroll
        for (int r = 0; r < 4; ++r)
          if (d + r < p.vdim) out[d + r] = BF16::from_float(o[i][4 * r4 + r] * f);
      }
    }
}

template <int NK, int NV, int MAPS>
static void go_prefill(const HeadAttnParams& p, hipStream_t s) {
  constexpr int smem = 2 * 4 * (NK + NV) * 32 * 16 * 2, kCols = 128 / MAPS;
  static_assert(MAPS == 1 || 64 * (32 * NV + 4) * 4 <= smem, "the second map's results take the place of the stages");
  if (smem > 64 * 1024)
    (void)hipFuncSetAttribute((const void*)head_prefill_kernel<NK, NV, MAPS>, hipFuncAttributeMaxDynamicSharedMemorySize, smem);
  const int64_t cols = (int64_t)p.max_query_len * (p.heads / p.kv_heads);
  hipLaunchKernelGGL((head_prefill_kernel<NK, NV, MAPS>),
                     dim3(p.kv_heads, (unsigned)((cols + kCols - 1) / kCols), p.num_seqs), dim3(256), smem, s, p);
}

template <int MAPS>
static int prefill_of_size(const HeadAttnParams& p, hipStream_t s) {
  LV_CHECK((int64_t)p.max_query_len * (p.heads / p.kv_heads) <= (int64_t)65535 * (128 / MAPS), "portion too long");
#define LV_HEAD_V(NK_)                               \
  switch (p.vpad / 32) {                             \
    case 1: go_prefill<NK_, 1, MAPS>(p, s); break;   \
    case 2: go_prefill<NK_, 2, MAPS>(p, s); break;   \
    case 3: go_prefill<NK_, 3, MAPS>(p, s); break;   \
    case 4: go_prefill<NK_, 4, MAPS>(p, s); break;   \
    case 6: go_prefill<NK_, 6, MAPS>(p, s); break;   \
    case 8: go_prefill<NK_, 8, MAPS>(p, s); break;   \
    default: LV_CHECK(false, "value size");          \
  }
  switch (p.kpad / 32) {
    case 2: LV_HEAD_V(2); break;
    case 3:
      if constexpr (MAPS == 1) { LV_HEAD_V(3); }
      else { LV_CHECK(false, "key size"); }
      break;
    case 4: LV_HEAD_V(4); break;
    case 6: LV_HEAD_V(6); break;
    case 8: LV_HEAD_V(8); break;
    default: LV_CHECK(false, "key size");
  }
#undef LV_HEAD_V
  LV_LAUNCH_CHECK();
  return 0;
}

}  // namespace lvllm
