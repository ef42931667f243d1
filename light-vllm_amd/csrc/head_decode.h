// The decode body of head_attention.h: single tokens, and portions so short that their (token, head) pairs fit the 16
// columns of one MFMA, over the paged cache.  With two maps a column is a (token, head, map) triple whose query is zero in the
// other map's half of the key.
//
// A workgroup serves one kv head of one sequence (and one share of its keys) for the whole GQA group from a single read
// of its keys and values: HBM-bound.  Wave w walks every fourth 16-key block of the share; blocks go straight into MFMA
// operands -- [kpad / 8][16][8] is the 16x16x32 A operand chunk by chunk, an 8-byte piece of a [vpad][16] row the
// 16x16x16 A operand -- with the next block's loads in flight.  The waves' results meet in LDS; shares meet in a second
// small launch, which also applies the gate and, with two maps, makes the difference.
#pragma once
#include <float.h>

#include "head_attention.h"

namespace lvllm {

template <int NK, int NV, int MAPS>
__global__ __launch_bounds__(256, 2) void head_decode_kernel(const HeadAttnParams p) {
  constexpr int KP = 32 * NK, VP = 32 * NV, NT = 2 * NV;
  extern __shared__ __attribute__((aligned(16))) char smem_raw[];
  float* so = reinterpret_cast<float*>(smem_raw);  // [4 waves][16 columns][VP + 4]
  __shared__ float sml[4][2][16];
  const int lane = threadIdx.x & 63;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int g = lane >> 4, c = lane & 15;
  const int G = p.heads / p.kv_heads * MAPS;  // (head, map) pairs of a kv head
  const int groups = (G + kDecodeCols - 1) / kDecodeCols;
  const int kvh = blockIdx.x / groups, cg = blockIdx.x - kvh * groups;
  const int seq = blockIdx.y, share = blockIdx.z;
  const int qbeg = p.query_start_loc[seq], qlen = p.query_start_loc[seq + 1] - qbeg;
  if (qlen <= 0 || qlen < p.min_query_len || !takes_decode_body(qlen, G)) return;
  const int seq_len = p.seq_lens[seq], ctx = seq_len - qlen;
  // columns of this workgroup
  int ncols, tok, head;
  if (qlen == 1) {
    ncols = min(kDecodeCols, G - cg * kDecodeCols);
    tok = 0;
    head = cg * kDecodeCols + min(c, ncols - 1);
  } else {
    if (cg > 0) return;
    ncols = qlen * G;
    const int cc = min(c, ncols - 1);
    tok = cc / G;
    head = cc - tok * G;
  }
  head += kvh * G;
  const int64_t row = qbeg + tok;
  const int pos = ctx + tok, low = first_seen(p, pos);
  const int first_block = first_seen(p, ctx) / 16;
  const int kept = min((p.keep_first + 15) / 16, first_block);  // blocks of kept keys ahead of the window's
  const int nblocks = (max(seq_len, 0) + 15) / 16 - first_block + kept;
  const int per = (nblocks + p.nsplit - 1) / p.nsplit;
  const int b0 = share * per, b1 = min(b0 + per, nblocks);
  auto block_of = [&](int b) { return b < kept ? b : b - kept + first_block; };

  h_u32x4_t qf[NK];
  {
    constexpr int HALF = NK / MAPS;
    const int map = MAPS == 2 ? head & 1 : 0;
    const uint16_t* q = (const uint16_t*)p.q + (row * (p.heads * MAPS) + head) * (KP / MAPS) + 8 * g;
#pragma unroll
    for (int j = 0; j < NK; ++j) {
      qf[j] = *reinterpret_cast<const h_u32x4_t*>(q + 32 * (j % HALF));
      if (MAPS == 2 && j / HALF != map) qf[j] = h_u32x4_t{0, 0, 0, 0};
    }
  }
  const int32_t* table = p.block_tables + (int64_t)seq * p.max_blocks;
  const uint16_t* kc = (const uint16_t*)p.k_cache + (int64_t)kvh * KP * 16 + lane * 8;
  const uint16_t* vc = (const uint16_t*)p.v_cache + (int64_t)kvh * VP * 16 + c * 16 + 4 * g;
  struct Tile {
    h_u32x4_t k[NK];
    uint2 v[NT];
  };
  auto fetch = [&](int b, Tile& t) __attribute__((always_inline)) {
    const int64_t blk = min(max(table[min(block_of(b), p.max_blocks - 1)], 0), p.max_block);
    const uint16_t* k = kc + blk * p.k_block_stride;
    const uint16_t* v = vc + blk * p.v_block_stride;
#pragma unroll
    for (int j = 0; j < NK; ++j) t.k[j] = *reinterpret_cast<const h_u32x4_t*>(k + j * 512);
#pragma unroll
    for (int j = 0; j < NT; ++j) t.v[j] = *reinterpret_cast<const uint2*>(v + j * 256);
  };
  const ScoreScale score(p);
  float m = -1e30f, l = 0.f;
  h_f32x4_t o[NT];
#pragma unroll
  for (int i = 0; i < NT; ++i) o[i] = h_f32x4_t{0.f, 0.f, 0.f, 0.f};
  auto use = [&](int b, const Tile& t) __attribute__((always_inline)) {
    h_f32x4_t s{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int j = 0; j < NK; ++j)
      s = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(h_bf16x8_t, t.k[j]),
                                                  __builtin_bit_cast(h_bf16x8_t, qf[j]), s, 0, 0, 0);
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int key = block_of(b) * 16 + 4 * g + r;
      const float z = score.cap > 0.f ? score.capped(s[r]) : s[r] * score.mul;
      s[r] = sees(p, key, pos, low) ? z : -FLT_MAX;
    }
    float mx = fmaxf(fmaxf(s[0], s[1]), fmaxf(s[2], s[3]));
    mx = fmaxf(mx, __shfl_xor(mx, 16));
    mx = fmaxf(mx, __shfl_xor(mx, 32));
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
    const uint2 pb{pack_bf16(s[0], s[1]), pack_bf16(s[2], s[3])};
    const h_s16x4_t pf = __builtin_bit_cast(h_s16x4_t, pb);
#pragma unroll
    for (int i = 0; i < NT; ++i)
      o[i] = __builtin_amdgcn_mfma_f32_16x16x16bf16_1k(__builtin_bit_cast(h_s16x4_t, t.v[i]), pf, o[i], 0, 0, 0);
  };
  Tile ta, tb;
  int b = b0 + wave;
  if (b < b1) fetch(b, ta);
  for (; b < b1; b += 8) {
    if (b + 4 < b1) fetch(b + 4, tb);
    use(b, ta);
    if (b + 4 >= b1) break;
    if (b + 8 < b1) fetch(b + 8, ta);
    use(b + 4, tb);
  }
  l += __shfl_xor(l, 16);
  l += __shfl_xor(l, 32);
  if (g == 0) {
    sml[wave][0][c] = m;
    sml[wave][1][c] = l;
  }
  __syncthreads();
  const float ma = fmaxf(fmaxf(sml[0][0][c], sml[1][0][c]), fmaxf(sml[2][0][c], sml[3][0][c]));
  const float corr = exp2f(m - ma);
  constexpr int LD = VP + 4;
#pragma unroll
  for (int i = 0; i < NT; ++i) {
    const h_f32x4_t v = o[i] * corr;
    *reinterpret_cast<h_f32x4_t*>(so + (wave * 16 + c) * LD + 16 * i + 4 * g) = v;
  }
  __syncthreads();
  for (int i = threadIdx.x; i < ncols * VP; i += 256) {
    const int cc = i / VP, d = i - cc * VP;
    int64_t r;
    int h;
    if (qlen == 1) {
      r = qbeg;
      h = kvh * G + cg * kDecodeCols + cc;
    } else {
      r = qbeg + cc / G;
      h = kvh * G + cc % G;
    }
    const float mm = fmaxf(fmaxf(sml[0][0][cc], sml[1][0][cc]), fmaxf(sml[2][0][cc], sml[3][0][cc]));
    const float ll = (sml[0][1][cc] * exp2f(sml[0][0][cc] - mm) + sml[1][1][cc] * exp2f(sml[1][0][cc] - mm)) +
                     (sml[2][1][cc] * exp2f(sml[2][0][cc] - mm) + sml[3][1][cc] * exp2f(sml[3][0][cc] - mm));
    const float v = (so[cc * LD + d] + so[(16 + cc) * LD + d]) + (so[(32 + cc) * LD + d] + so[(48 + cc) * LD + d]);
    if (MAPS == 2 || p.nsplit > 1) {
      const int64_t at = (r * (p.heads * MAPS) + h) * p.nsplit + share;
      p.part_o[at * VP + d] = v;
      if (d == 0) {
        p.part_ml[2 * at] = mm;
        p.part_ml[2 * at + 1] = ll;
      }
    } else if (d < p.vdim) {
      const float w = ll > 0.f ? v / (ll + sink_term(p, h, mm)) * gate_of<BF16>(p, r, h) : 0.f;
      ((uint16_t*)p.out)[r * p.out_stride + (int64_t)h * p.vdim + d] = BF16::from_float(w);
    }
  }
}

// Shares of one (row, head) -> out, gate applied.  Rows of sequences that took the chunk body are left alone.
template <int MAPS>
__global__ __launch_bounds__(128) void head_decode_reduce_kernel(const HeadAttnParams p) {
  const int row = blockIdx.x, head = blockIdx.y;
  const int seq = find_seq(p.query_start_loc, p.num_seqs, row);
  if (seq >= p.num_seqs) return;
  const int qlen = p.query_start_loc[seq + 1] - p.query_start_loc[seq];
  if (qlen < p.min_query_len || !takes_decode_body(qlen, p.heads / p.kv_heads * MAPS)) return;
  // the shares' weights, one share per lane (nsplit <= 64), through LDS
  __shared__ float weight[MAPS][64];
  const int64_t at = ((int64_t)row * p.heads + head) * MAPS * p.nsplit;
  const int lane = threadIdx.x & 63;
#pragma unroll
  for (int i = 0; i < MAPS; ++i) {
    const float2 ml = lane < p.nsplit ? *reinterpret_cast<const float2*>(p.part_ml + 2 * (at + i * p.nsplit + lane)) : float2{-1e30f, 0.f};
    const float m = wave_max(ml.x), w = lane < p.nsplit ? exp2f(ml.x - m) : 0.f, l = wave_sum(ml.y * w);
    weight[i][lane] = l > 0.f ? w / (l + sink_term(p, head, m)) : 0.f;
  }
  __syncthreads();
  auto sum_of = [&](int i, int d) __attribute__((always_inline)) {
    constexpr int B = 8;  // loads in flight
    const float* part = p.part_o + (at + i * p.nsplit) * p.vpad + d;
    float v = 0.f;
    for (int s0 = 0; s0 < p.nsplit; s0 += B) {
      float t[B];
#pragma unroll
      for (int s = 0; s < B; ++s) t[s] = part[(int64_t)min(s0 + s, p.nsplit - 1) * p.vpad];
#pragma unroll
      for (int s = 0; s < B; ++s)
        if (s0 + s < p.nsplit) v = fmaf(t[s], weight[i][s0 + s], v);
    }
    return v;
  };
  uint16_t* out = (uint16_t*)p.out + row * p.out_stride + (int64_t)head * p.vdim;
  const float gate = gate_of<BF16>(p, row, head);
  if constexpr (MAPS == 1) {
    for (int d = threadIdx.x; d < p.vdim; d += 128) out[d] = BF16::from_float(sum_of(0, d) * gate);
  } else {
    __shared__ float red[16];
    float v[2], ss = 0.f;  // (vdim <= 256)
#pragma unroll
    for (int j = 0; j < 2; ++j) {
      const int d = threadIdx.x + 128 * j;
      v[j] = d < p.vdim ? fmaf(-p.map_weight, sum_of(1, d), sum_of(0, d)) : 0.f;
      ss = fmaf(v[j], v[j], ss);
    }
    const float n = gate / sqrtf(block_sum(ss, red) / (float)p.vdim + p.map_eps);
#pragma unroll
    for (int j = 0; j < 2; ++j)
      if ((int)threadIdx.x + 128 * j < p.vdim) out[threadIdx.x + 128 * j] = BF16::from_float(v[j] * n);
  }
}

template <int NK, int NV, int MAPS>
static void go_decode(const HeadAttnParams& p, hipStream_t s) {
  constexpr int smem = 4 * 16 * (32 * NV + 4) * 4;
  if (smem > 64 * 1024)
    (void)hipFuncSetAttribute((const void*)head_decode_kernel<NK, NV, MAPS>, hipFuncAttributeMaxDynamicSharedMemorySize, smem);
  const int groups = (p.heads / p.kv_heads * MAPS + kDecodeCols - 1) / kDecodeCols;
  hipLaunchKernelGGL((head_decode_kernel<NK, NV, MAPS>), dim3(p.kv_heads * groups, p.num_seqs, p.nsplit), dim3(256), smem, s, p);
}

template <int MAPS>
static int decode_of_size(const HeadAttnParams& p, hipStream_t s) {
#define LV_HEAD_V(NK_)                              \
  switch (p.vpad / 32) {                            \
    case 1: go_decode<NK_, 1, MAPS>(p, s); break;   \
    case 2: go_decode<NK_, 2, MAPS>(p, s); break;   \
    case 3: go_decode<NK_, 3, MAPS>(p, s); break;   \
    case 4: go_decode<NK_, 4, MAPS>(p, s); break;   \
    case 6: go_decode<NK_, 6, MAPS>(p, s); break;   \
    case 8: go_decode<NK_, 8, MAPS>(p, s); break;   \
    default: LV_CHECK(false, "value size");         \
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
  if (MAPS == 2 || p.nsplit > 1) {
    hipLaunchKernelGGL((head_decode_reduce_kernel<MAPS>), dim3(p.rows, p.heads), dim3(128), 0, s, p);
    LV_LAUNCH_CHECK();
  }
  return 0;
}

}  // namespace lvllm
