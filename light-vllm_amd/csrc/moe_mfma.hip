// The products of moe.h on 16x16x32 bf16 MFMAs over packed weights: W rows are the A operand, slots the columns, so that a
// lane ends up with consecutive outputs of one slot, and gate and value of an activation in the same register of two tiles.
//
//   * few slots per expert (decode steps): bound by the weights' bytes.  A workgroup takes 16 slots of one expert and a share
//     of its outputs; the slots' rows sit in LDS in fragment order (2048 of K at a time), every wave streams the two W tiles
//     of its own (1 KiB a load, eight k-steps in flight behind the eight in use) and needs no other wave;
//   * prompts: 256 W rows x 128 slots a workgroup, a wave 64 x 128.  W goes from memory straight into the operand registers
//     of the one wave that uses it, the slots' rows straight to LDS, 32 of K a step, three steps in flight behind the one in
//     use (through LDS, W would take more of its bandwidth than there is).  A slot's 64 bytes are four chunks, exchanged so
//     that a fragment read is free of bank conflicts.  An XCD gets consecutive work: up to eight tiles of an expert side by
//     side, W block after W block, so that its L2 serves a W block to all of them and their rows to the next blocks.
#include "moe.h"

namespace lvllm {

typedef __bf16 e_bf16x8_t __attribute__((ext_vector_type(8)));
typedef float e_f32x4_t __attribute__((ext_vector_type(4)));
typedef unsigned int e_u32x4_t __attribute__((ext_vector_type(4)));

__device__ __forceinline__ e_f32x4_t moe_mfma(e_u32x4_t a, e_u32x4_t b, e_f32x4_t c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(e_bf16x8_t, a), __builtin_bit_cast(e_bf16x8_t, b), c, 0, 0,
                                                 0);
}

constexpr int kStreamBatch = 8, kStreamChunk = 64;  // k-steps per batch, per LDS chunk

// grid (shares of the outputs, tiles of 16 slots); a wave computes W tiles 2 u and 2 u + 1, or (KS > 1, when few
// experts have work) a KS-th of their k-steps, 64 / KS of every LDS chunk
template <int PRODUCT, int KS>
__global__ __launch_bounds__(256, 2) void moe_stream_kernel(const MoeParams p) {
  constexpr bool UP = PRODUCT != kMoeDown, GATED = PRODUCT == kMoeGated;
  extern __shared__ __attribute__((aligned(16))) char sx[];  // [k-steps of a chunk][4][16][8]
  __shared__ e_f32x4_t red[KS > 1 ? 4 : 1][2][64];
  const int e = p.tiles[4 * blockIdx.y];
  if (e < 0 || e >= p.experts) return;
  const int s0 = p.tiles[4 * blockIdx.y + 1], s1 = min(min(p.offsets[e + 1], s0 + 16), p.slots);
  if (s0 >= s1) return;
  const int lane = threadIdx.x & 63;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int g = lane >> 4, c = lane & 15;
  const int ff = p.ff[e], K = UP ? p.width : ff, steps = K >> 5;
  const int units = GATED ? ff >> 4 : (UP ? ff : p.width) >> 5;
  constexpr int U = 4 / KS, P = kStreamChunk / KS;  // units of a workgroup; this wave's k-steps of a chunk
  if ((int)blockIdx.x * U >= units) return;
  const int u = min((int)blockIdx.x * U + wave / KS, units - 1), kq = wave % KS;  // (a wave too many repeats the last unit)
  // k-steps, some missing ones of the last chunk included
  const int mine = KS == 1 ? (steps + 2 * kStreamBatch - 1) / (2 * kStreamBatch) * (2 * kStreamBatch)
                           : (steps + kStreamChunk - 1) / kStreamChunk * P;
  auto step_of = [&](int v) { return KS == 1 ? v : v / P * kStreamChunk + kq * P + v % P; };  // of batch v, a multiple of 8
  const uint16_t* w = (const uint16_t*)p.w + p.w_offset[e] + (int64_t)2 * u * steps * 512 + lane * 8;
  e_u32x4_t a[2][2][kStreamBatch];
  auto fetch = [&](int v, e_u32x4_t (&t)[2][kStreamBatch]) __attribute__((always_inline)) {
    const int b = step_of(v);
#pragma unroll
    for (int j = 0; j < kStreamBatch; ++j)
#pragma unroll
      for (int i = 0; i < 2; ++i)  // (a missing step: the last one again)
        t[i][j] = *reinterpret_cast<const e_u32x4_t*>(w + ((int64_t)i * steps + min(b + j, steps - 1)) * 512);
  };
  fetch(0, a[0]);
  const int64_t ld = UP ? p.width : p.ff_max;
  const int my_slot = s0 + (threadIdx.x & 15);
  const int64_t row = my_slot >= s1 ? -1 : UP ? min(max(p.token[my_slot], 0), p.rows - 1) : my_slot;
  const uint16_t* x = (const uint16_t*)p.x + (row < 0 ? 0 : row) * ld;
  auto stage = [&](int step0) __attribute__((always_inline)) {
    const int n = min(kStreamChunk, steps - step0) * 64;
    for (int i = threadIdx.x; i < n; i += 256) {  // 16-byte chunk i: slot i % 16, entries 8 (i / 16) ..
      e_u32x4_t v{0, 0, 0, 0};
      if (row >= 0) v = *reinterpret_cast<const e_u32x4_t*>(x + step0 * 32 + (i >> 4) * 8);
      *reinterpret_cast<e_u32x4_t*>(sx + i * 16) = v;
    }
    __syncthreads();
  };
  const char* xf = sx + lane * 16;
  e_f32x4_t acc[2] = {e_f32x4_t{0.f, 0.f, 0.f, 0.f}, e_f32x4_t{0.f, 0.f, 0.f, 0.f}};
  auto use = [&](int v, const e_u32x4_t (&t)[2][kStreamBatch]) __attribute__((always_inline)) {
    const int b = step_of(v), at = b % kStreamChunk;
    auto one = [&](int j) __attribute__((always_inline)) {
      const e_u32x4_t xv = *reinterpret_cast<const e_u32x4_t*>(xf + (at + j) * 1024);
      acc[0] = moe_mfma(t[0][j], xv, acc[0]);
      acc[1] = moe_mfma(t[1][j], xv, acc[1]);
    };
    if (b + kStreamBatch <= steps) {
#pragma unroll
      for (int j = 0; j < kStreamBatch; ++j) one(j);
    } else {
#pragma unroll
      for (int j = 0; j < kStreamBatch; ++j)
        if (b + j < steps) one(j);
    }
  };
  stage(0);
  for (int v = 0; v < mine; v += 2 * kStreamBatch) {
    fetch(v + kStreamBatch, a[1]);
    if (v > 0 && v % P == 0) {
      __syncthreads();
      stage(v / P * kStreamChunk);
    }
    use(v, a[0]);
    fetch(v + 2 * kStreamBatch, a[0]);
    use(v + kStreamBatch, a[1]);
  }
  if constexpr (KS > 1) {
    red[wave][0][lane] = acc[0];
    red[wave][1][lane] = acc[1];
    __syncthreads();
    if (kq != 0 || (int)blockIdx.x * U + wave / KS >= units) return;
#pragma unroll
    for (int i = 0; i < 2; ++i)
#pragma unroll
      for (int q = 1; q < KS; ++q) acc[i] += red[wave + q][i][lane];
  }
  const int slot = s0 + c;
  if (slot >= s1) return;
  float v[4];
  const float f = UP ? slot_weight_of(p, slot) : 1.f;
  if constexpr (GATED) {
    const MoeActivation act(p, e);
#pragma unroll
    for (int r = 0; r < 4; ++r) v[r] = act(acc[0][r] * f, acc[1][r] * f);
    store4<BF16>((uint16_t*)p.out + (int64_t)slot * p.ff_max + 16 * u + 4 * g, v);
  } else {
#pragma unroll
    for (int i = 0; i < 2; ++i) {
#pragma unroll
      for (int r = 0; r < 4; ++r) v[r] = UP ? relu_squared_of(acc[i][r] * f) : acc[i][r];
      store4<BF16>((uint16_t*)p.out + (int64_t)slot * (UP ? p.ff_max : p.width) + 32 * u + 16 * i + 4 * g, v);
    }
  }
}

constexpr int kTileW = 16;                                 // W tiles of a workgroup
constexpr int kStages = 4, kStageBytes = kMoeTile * 64;    // of 32 of K: 16-slot groups of 1 KiB

__device__ __forceinline__ void to_lds(const uint16_t* src, char* dst) {  // 16 bytes a lane, 1 KiB a wave
  __builtin_amdgcn_global_load_lds((const __attribute__((address_space(1))) void*)src,
                                   (__attribute__((address_space(3))) void*)dst, 16, 0, 0);
}

template <int PRODUCT>
__global__ __launch_bounds__(256, 2) void moe_tile_kernel(const MoeParams p, const int blocks_first, const int blocks_last) {
  constexpr bool UP = PRODUCT != kMoeDown, GATED = PRODUCT == kMoeGated;
  __shared__ __attribute__((aligned(16))) char ring[kStages][kStageBytes];
  // the tiles of all experts but the last one, then the last one's (the shared expert may be larger): an eighth of each to
  // every XCD
  const int tiles_first = p.tiles[4 * p.max_tiles], tiles_all = p.tiles[4 * p.max_tiles + 1];
  const int xcd = blockIdx.x & 7, turn = blockIdx.x >> 3;
  const int all_first = tiles_first * blocks_first, all_last = (tiles_all - tiles_first) * blocks_last;
  const int per_first = (all_first + 7) / 8, per_last = (all_last + 7) / 8;
  int unit, blocks, tile;
  if (turn < per_first) {
    unit = xcd * per_first + turn;
    if (unit >= all_first) return;
    blocks = blocks_first;
    tile = unit / blocks;
  } else {
    unit = xcd * per_last + turn - per_first;
    if (turn - per_first >= per_last || unit >= all_last) return;
    blocks = blocks_last;
    tile = tiles_first + unit / blocks;
    unit += tiles_first * blocks;
  }
  constexpr int kSide = 8;
  const int e = p.tiles[4 * tile], tile0 = p.tiles[4 * tile + 2], count = p.tiles[4 * tile + 3];
  if (e < 0 || e >= p.experts || count <= 0) return;
  unit -= tile0 * blocks;  // of this expert's
  const int group = unit / (kSide * blocks), side = min(kSide, count - group * kSide);
  unit -= group * kSide * blocks;
  const int block = unit / side;
  tile = tile0 + group * kSide + unit - block * side;
  const int s0 = p.tiles[4 * tile + 1], s1 = min(min(p.offsets[e + 1], s0 + kMoeTile), p.slots);
  const int ff = p.ff[e], steps = (UP ? p.width : ff) >> 5;
  const int ntiles = GATED ? ff >> 3 : (UP ? ff : p.width) >> 4;  // of 16 W rows
  if (block * kTileW >= ntiles || s0 >= s1) return;
  const int lane = threadIdx.x & 63;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int g = lane >> 4, c = lane & 15;
  const int64_t ld = UP ? p.width : p.ff_max;
  const int nt0 = block * kTileW + wave * 4;
  // this wave's W tiles, and the two 16-slot groups it copies: lane l moves chunk l % 4, exchanged by slot / 4, of slot l / 4
  const uint16_t *wsrc[4], *xsrc[2];
  const uint16_t* w = (const uint16_t*)p.w + p.w_offset[e] + lane * 8;
#pragma unroll
  for (int j = 0; j < 4; ++j) wsrc[j] = w + (int64_t)min(nt0 + j, ntiles - 1) * steps * 512;
#pragma unroll
  for (int j = 0; j < 2; ++j) {
    const int slot = min(s0 + (wave * 2 + j) * 16 + (lane >> 2), s1 - 1);
    const int64_t row = UP ? min(max(p.token[slot], 0), p.rows - 1) : slot;
    xsrc[j] = (const uint16_t*)p.x + row * ld + ((lane & 3) ^ (lane >> 4)) * 8;
  }
  e_u32x4_t a[kStages][4];
  auto issue = [&](int k, int stage) __attribute__((always_inline)) {  // (past the end: the last step once more)
    k = min(k, steps - 1);
#pragma unroll
    for (int j = 0; j < 2; ++j) to_lds(xsrc[j] + k * 32, ring[stage] + (wave * 2 + j) * 1024);
#pragma unroll
    for (int j = 0; j < 4; ++j) a[stage][j] = *reinterpret_cast<const e_u32x4_t*>(wsrc[j] + k * 512);
  };
  constexpr int MT = kMoeTile / 16;
  const int xoff = c * 64 + ((g ^ (c >> 2)) * 16);
  e_f32x4_t acc[4][MT];
#pragma unroll
  for (int n = 0; n < 4; ++n)
#pragma unroll
    for (int m = 0; m < MT; ++m) acc[n][m] = e_f32x4_t{0.f, 0.f, 0.f, 0.f};
  auto step = [&](int k, int stage) __attribute__((always_inline)) {
    // loads retire in order: with only the two younger steps' six each outstanding, this one's have landed
    __builtin_amdgcn_s_waitcnt(12 | (7 << 4) | (15 << 8));
    asm volatile("s_barrier" ::: "memory");  // ... for every wave; and everyone is done with the stage that is filled next
    issue(k + 3, (stage + 3) % kStages);
    e_u32x4_t x[MT];
#pragma unroll
    for (int m = 0; m < MT; ++m) x[m] = *reinterpret_cast<const e_u32x4_t*>(ring[stage] + xoff + m * 1024);
    __builtin_amdgcn_sched_barrier(0);
#pragma unroll
    for (int m = 0; m < MT; ++m)
#pragma unroll
      for (int n = 0; n < 4; ++n) acc[n][m] = moe_mfma(a[stage][n], x[m], acc[n][m]);
  };
  issue(0, 0);
  issue(1, 1);
  issue(2, 2);
  int k = 0;
  for (; k + 4 <= steps; k += 4) {
    step(k, 0);
    step(k + 1, 1);
    step(k + 2, 2);
    step(k + 3, 3);
  }
  if (k < steps) step(k, 0);
  if (k + 1 < steps) step(k + 1, 1);
  if (k + 2 < steps) step(k + 2, 2);
  __builtin_amdgcn_s_waitcnt(0 | (7 << 4) | (15 << 8));  // (no copy to LDS outlives the workgroup)
  [[maybe_unused]] const MoeActivation act(p, GATED ? e : -1);
#pragma unroll
  for (int m = 0; m < MT; ++m) {
    const int slot = s0 + 16 * m + c;
    if (slot >= s1) continue;
    const float f = UP ? slot_weight_of(p, slot) : 1.f;
#pragma unroll
    for (int n = 0; n < 4; n += GATED ? 2 : 1) {
      if (nt0 + n >= ntiles) continue;
      float v[4];
      if constexpr (GATED) {
#pragma unroll
        for (int r = 0; r < 4; ++r) v[r] = act(acc[n][m][r] * f, acc[n + 1][m][r] * f);
        store4<BF16>((uint16_t*)p.out + (int64_t)slot * p.ff_max + (nt0 + n) * 8 + 4 * g, v);
      } else {
#pragma unroll
        for (int r = 0; r < 4; ++r) v[r] = UP ? relu_squared_of(acc[n][m][r] * f) : acc[n][m][r];
        store4<BF16>((uint16_t*)p.out + (int64_t)slot * (UP ? p.ff_max : p.width) + (nt0 + n) * 16 + 4 * g, v);
      }
    }
  }
}

// The router's logits on packed weights (experts and the shared gate, up to a multiple of 16 rows): 16 rows of h and a share
// of the k-steps a workgroup; its 8 waves take every eighth step of eight tiles of weights and meet in LDS in wave order.
// z [rows 16 at a time][ld] in LDS, without the bias.
constexpr int kRouteTiles = 8, kRouteBatch = 4;  // tiles and k-steps in flight
constexpr int kRouteShares = 16;              // most shares of the k-steps
constexpr int kRouteLds = 8 * kRouteTiles * 1024;

__device__ __forceinline__ void route_logits(float* z, int ld, e_f32x4_t* red, const uint16_t* h, const uint16_t* w, int row0,
                                             int rows, int width, int ntiles, int step0, int step1) {
  constexpr int TG = kRouteTiles, B = kRouteBatch;
  const int lane = threadIdx.x & 63;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int g = lane >> 4, c = lane & 15, steps = width >> 5;
  const uint16_t* x = h + (int64_t)min(row0 + c, rows - 1) * width + 8 * g;
  for (int t0 = 0; t0 < ntiles; t0 += TG) {
    e_f32x4_t acc[TG];
#pragma unroll
    for (int i = 0; i < TG; ++i) acc[i] = e_f32x4_t{0.f, 0.f, 0.f, 0.f};
    for (int k0 = step0 + wave; k0 < step1; k0 += 8 * B) {
      e_u32x4_t xv[B], wv[B][TG];
#pragma unroll
      for (int j = 0; j < B; ++j) {
        const int k = min(k0 + 8 * j, step1 - 1);
        xv[j] = k0 + 8 * j < step1 ? *reinterpret_cast<const e_u32x4_t*>(x + 32 * k) : e_u32x4_t{0, 0, 0, 0};
#pragma unroll
        for (int i = 0; i < TG; ++i)
          if (t0 + i < ntiles) wv[j][i] = *reinterpret_cast<const e_u32x4_t*>(w + ((int64_t)(t0 + i) * steps + k) * 512 + lane * 8);
      }
#pragma unroll
      for (int i = 0; i < TG; ++i)
        if (t0 + i < ntiles) {
#pragma unroll
          for (int j = 0; j < B; ++j) acc[i] = moe_mfma(wv[j][i], xv[j], acc[i]);
        }
    }
#pragma unroll
    for (int i = 0; i < TG; ++i) red[(wave * TG + i) * 64 + lane] = acc[i];
    __syncthreads();
    if (t0 + wave < ntiles) {  // wave i sums tile i
      e_f32x4_t s = red[threadIdx.x];
#pragma unroll
      for (int v = 1; v < 8; ++v) s += red[v * TG * 64 + threadIdx.x];
#pragma unroll
      for (int r = 0; r < 4; ++r) z[c * ld + (t0 + wave) * 16 + 4 * g + r] = s[r];
    }
    __syncthreads();
  }
}

// many rows: logits and choice in one launch, a wave chooses for two rows
__global__ __launch_bounds__(512) void moe_route_mfma_kernel(int32_t* ids, float* __restrict__ weights,
                                                             const uint16_t* __restrict__ h, const uint16_t* __restrict__ w,
                                                             const float* __restrict__ bias, const MoeRouting r,
                                                             const int rows, const int width, const MoeGroups groups) {
  extern __shared__ __attribute__((aligned(16))) char smem[];
  float* z = reinterpret_cast<float*>(smem + kRouteLds);
  const int ntiles = (r.logits() + 15) >> 4, ld = ntiles * 16 + 1, row0 = blockIdx.x * 16, n = r.per_row();
  route_logits(z, ld, reinterpret_cast<e_f32x4_t*>(smem), h, w, row0, rows, width, ntiles, 0, width >> 5);
  const int lane = threadIdx.x & 63;
  for (int i = threadIdx.x >> 6; i < 16 && row0 + i < rows; i += 8) {
    if (bias != nullptr)
      for (int e = lane; e < r.experts; e += 64) z[i * ld + e] += bias[e];
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");  // (the wave's own next reads see it)
    choose_experts(z + i * ld, r, ids + (int64_t)(row0 + i) * n, weights + (int64_t)(row0 + i) * n);
  }
  __syncthreads();  // (the logits' partial sums make room for the counts)
  moe_count_assignments(ids, row0, min(16, rows - row0), n, r.all(), r.shared, reinterpret_cast<int*>(smem), groups);
}

__global__ __launch_bounds__(256) void moe_zero_kernel(int32_t* __restrict__ p, const int n) {
  for (int i = threadIdx.x; i < n; i += 256) p[i] = 0;
}

// few rows: the k-steps are dealt to workgroups as well (grid.y), whose logits leave as part [share][16-row tiles][16][ld]
__global__ __launch_bounds__(512) void moe_logits_kernel(float* __restrict__ part, const uint16_t* __restrict__ h,
                                                         const uint16_t* __restrict__ w, const int ntiles, const int rows,
                                                         const int width, const int per) {
  extern __shared__ __attribute__((aligned(16))) char smem[];
  float* z = reinterpret_cast<float*>(smem + kRouteLds);
  const int ld = ntiles * 16, step0 = blockIdx.y * per, step1 = min(step0 + per, width >> 5);
  route_logits(z, ld, reinterpret_cast<e_f32x4_t*>(smem), h, w, blockIdx.x * 16, rows, width, ntiles, step0, step1);
  float* out = part + ((int64_t)blockIdx.y * gridDim.x + blockIdx.x) * 16 * ld;
  for (int i = threadIdx.x; i < 16 * ld; i += 512) out[i] = z[i];
}

// ... and one workgroup adds them, chooses (a wave per row) and groups the assignments
__global__ __launch_bounds__(1024) void moe_choose_group_kernel(int32_t* ids, float* weights, const float* __restrict__ part,
                                                                const float* __restrict__ bias, const int shares,
                                                                const int row_tiles, const int ld, const MoeRouting r,
                                                                const int rows, const MoeGroups groups) {
  extern __shared__ __attribute__((aligned(16))) char smem[];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, n = r.per_row();
  float* z = reinterpret_cast<float*>(smem) + wave * ld;
  for (int row = wave; row < rows; row += 16) {
    for (int e = lane; e < r.logits(); e += 64) {
      float v = e < r.experts && bias != nullptr ? bias[e] : 0.f, t[kRouteShares];
#pragma unroll
      for (int s = 0; s < kRouteShares; ++s) t[s] = part[((int64_t)min(s, shares - 1) * row_tiles * 16 + row) * ld + e];
#pragma unroll
      for (int s = 0; s < kRouteShares; ++s) v += s < shares ? t[s] : 0.f;
      z[e] = v;
    }
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");  // (the wave's own next reads see it)
    choose_experts(z, r, ids + (int64_t)row * n, weights + (int64_t)row * n);
  }
  __syncthreads();
  group_assignments(ids, rows * n, n, r.all(), r.shared, groups);
}

static int route_shares(int width) {
  const int steps = width / 32;
  return steps < 16 ? 1 : steps / 16 > kRouteShares ? kRouteShares : steps / 16;  // (at least two k-steps a wave)
}

int64_t moe_route_mfma_workspace(const MoeRouting& r, int rows, int width) {
  if (rows > kMoeFewRows) return (int64_t)r.all() * 4;  // (the experts' counts)
  return (int64_t)route_shares(width) * ((rows + 15) / 16) * 16 * ((r.logits() + 15) / 16 * 16) * 4;
}

int launch_moe_route_mfma(int32_t* ids, float* weights, const void* h, const void* w, const float* bias, const MoeRouting& r,
                          int rows, int width, const MoeGroups& groups, float* workspace, hipStream_t s) {
  const int ntiles = (r.logits() + 15) / 16, row_tiles = (rows + 15) / 16;
  if (rows <= kMoeFewRows) {
    const int shares = route_shares(width), per = (width / 32 + shares - 1) / shares, ld = ntiles * 16;
    const int lds = kRouteLds + 16 * ld * 4, lds_choose = 16 * ld * 4;
    (void)hipFuncSetAttribute((const void*)moe_logits_kernel, hipFuncAttributeMaxDynamicSharedMemorySize, lds);
    (void)hipFuncSetAttribute((const void*)moe_choose_group_kernel, hipFuncAttributeMaxDynamicSharedMemorySize, lds_choose);
    hipLaunchKernelGGL(moe_logits_kernel, dim3(row_tiles, shares), dim3(512), lds, s, workspace, (const uint16_t*)h,
                       (const uint16_t*)w, ntiles, rows, width, per);
    LV_LAUNCH_CHECK();
    hipLaunchKernelGGL(moe_choose_group_kernel, dim3(1), dim3(1024), lds_choose, s, ids, weights, workspace, bias, shares,
                       row_tiles, ld, r, rows, groups);
    LV_LAUNCH_CHECK();
    return 0;
  }
  const int lds = kRouteLds + 16 * (ntiles * 16 + 1) * 4;
  (void)hipFuncSetAttribute((const void*)moe_route_mfma_kernel, hipFuncAttributeMaxDynamicSharedMemorySize, lds);
  hipLaunchKernelGGL(moe_zero_kernel, dim3(1), dim3(256), 0, s, groups.count, r.all());
  LV_LAUNCH_CHECK();
  hipLaunchKernelGGL(moe_route_mfma_kernel, dim3(row_tiles), dim3(512), lds, s, ids, weights, (const uint16_t*)h,
                     (const uint16_t*)w, bias, r, rows, width, groups);
  LV_LAUNCH_CHECK();
  return launch_moe_group(ids, rows * r.per_row(), r.per_row(), r.all(), r.shared, true, groups, s);
}

bool moe_takes_mfma(int width, int dtype) { return dtype == LVLLM_BF16 && width % 32 == 0; }

template <int PRODUCT>
static void go(const MoeParams& p, hipStream_t s) {
  constexpr bool UP = PRODUCT != kMoeDown, GATED = PRODUCT == kMoeGated;
  if (p.rows <= kMoeFewRows) {
    const int steps = (UP ? p.width : p.ff_max) / 32;  // of the largest expert
    const int units = GATED ? p.ff_max / 16 : (UP ? p.ff_max : p.width) / 32;
    const int smem = (steps < kStreamChunk ? steps : kStreamChunk) * 1024;
    // workgroups with work, were every wave to take whole units
    const int64_t wgs = (int64_t)p.max_tiles * (((GATED ? p.ff_first / 16 : UP ? p.ff_first / 32 : units) + 3) / 4);
    const unsigned t = p.max_tiles;
    if (wgs <= 256) hipLaunchKernelGGL((moe_stream_kernel<PRODUCT, 4>), dim3(units, t), dim3(256), smem, s, p);
    else if (wgs <= 512) hipLaunchKernelGGL((moe_stream_kernel<PRODUCT, 2>), dim3((units + 1) / 2, t), dim3(256), smem, s, p);
    else hipLaunchKernelGGL((moe_stream_kernel<PRODUCT, 1>), dim3((units + 3) / 4, t), dim3(256), smem, s, p);
  } else {
    auto blocks = [&](int ff) { return ((GATED ? ff / 8 : (UP ? ff : p.width) / 16) + kTileW - 1) / kTileW; };
    const int first = blocks(p.ff_first), last = blocks(p.ff_last);
    const int64_t last_tiles = (p.rows + kMoeTile - 1) / kMoeTile;  // a token takes an expert once
    const int64_t wgs = 8 * (((int64_t)p.max_tiles * first + 7) / 8 + (last_tiles * last + 7) / 8);
    hipLaunchKernelGGL((moe_tile_kernel<PRODUCT>), dim3((unsigned)wgs), dim3(256), 0, s, p, first, last);
  }
}

int launch_moe_mfma(const MoeParams& p, int product, hipStream_t s) {
  LV_CHECK(p.experts <= 65535 && p.ff_first > 0 && p.ff_last > 0 && p.ff_first <= p.ff_max && p.ff_last <= p.ff_max,
           "sizes of the experts");
  if (product == kMoeGated) go<kMoeGated>(p, s);
  else if (product == kMoePlain) go<kMoePlain>(p, s);
  else go<kMoeDown>(p, s);
  LV_LAUNCH_CHECK();
  return 0;
}

}  // namespace lvllm
