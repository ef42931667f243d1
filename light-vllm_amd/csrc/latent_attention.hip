// Latent attention: the cache write, queries into latent space, the gather and the expansion for long portions, and the plain
// attention body with its values' way out of latent space (see latent_attention.h for the layouts).
#include <float.h>

#include "latent_attention.h"

namespace lvllm {

typedef __bf16 l_bf16x8_t __attribute__((ext_vector_type(8)));
typedef float l_f32x4_t __attribute__((ext_vector_type(4)));

struct LatentCacheParams {
  void* cache;
  const void* kv;          // null: nothing to write
  const float* weight;
  const int64_t *positions, *slot_mapping;
  const double* turns;
  int64_t block_stride, num_slots, kv_stride;
  int block_size, cpad, rpad, kv_rank, rot_dim, rot_dims, rows;
  float eps, grow;  // grow: of the rotation
};

// RMS-normed latent and rotated key part of a row -> its cache slot; one wave, 16 bytes a lane where the sizes allow it
template <typename T>
__device__ __forceinline__ void write_latent_row(const LatentCacheParams& p, int row) {
  using S = typename T::store_t;
  constexpr int X = 16 / sizeof(S);
  const int lane = threadIdx.x & 63;
  const S* z = (const S*)p.kv + row * p.kv_stride;
  const bool vec = p.kv_rank % X == 0 && p.kv_rank <= 64 * X && ((uintptr_t)z & 15) == 0;
  const int64_t wide = p.slot_mapping[row], pos = p.positions[row];
  Vec16<T> raw{};
  float weight[X];
#pragma unroll
  for (int j = 0; j < X; ++j) weight[j] = 0.f;
  if (vec && lane * X < p.kv_rank) {  // (asked for before the slot is known)
    raw = *reinterpret_cast<const Vec16<T>*>(z + lane * X);
#pragma unroll
    for (int j = 0; j < X; ++j) weight[j] = p.weight[lane * X + j];
  }
  if (wide < 0 || wide >= p.num_slots) return;
  const unsigned slot = (unsigned)wide, block = slot / (unsigned)p.block_size;
  S* out = (S*)p.cache + block * p.block_stride + (slot - block * p.block_size) * (int64_t)(p.cpad + p.rpad);
  float ss = 0.f;
  if (vec) {
    float v[X];
#pragma unroll
    for (int j = 0; j < X; ++j) {
      v[j] = T::to_float(raw.v[j]);
      ss = fmaf(v[j], v[j], ss);
    }
    const float f = 1.f / sqrtf(wave_sum(ss) / (float)p.kv_rank + p.eps);
    if (lane * X < p.cpad) {
#pragma unroll
      for (int j = 0; j < X; ++j) raw.v[j] = T::from_float(v[j] * f * weight[j]);
      *reinterpret_cast<Vec16<T>*>(out + lane * X) = raw;
    }
    for (int d = 64 * X + lane; d < p.cpad; d += 64) out[d] = T::from_float(0.f);
  } else {
    for (int i = lane; i < p.kv_rank; i += 64) {
      const float v = T::to_float(z[i]);
      ss = fmaf(v, v, ss);
    }
    const float f = 1.f / sqrtf(wave_sum(ss) / (float)p.kv_rank + p.eps);
    for (int i = lane; i < p.cpad; i += 64) out[i] = T::from_float(i < p.kv_rank ? T::to_float(z[i]) * f * p.weight[i] : 0.f);
  }
  z += p.kv_rank;
  out += p.cpad;
  for (int i = lane * 2; i < p.rpad; i += 128) {
    float u = i < p.rot_dim ? T::to_float(z[i]) : 0.f, v = i + 1 < p.rot_dim ? T::to_float(z[i + 1]) : 0.f;
    if (i < p.rot_dims) {
      float c, s;
      rotation_of(pos, p.turns[i >> 1], p.grow, c, s);
      const float t = u * c - v * s;
      v = v * c + u * s;
      u = t;
    }
    out[i] = T::from_float(u);
    out[i + 1] = T::from_float(v);
  }
}

template <typename T>
__global__ __launch_bounds__(256) void latent_cache_kernel(const LatentCacheParams p) {
  const int row = blockIdx.x * 4 + (threadIdx.x >> 6);
  if (row < p.rows) write_latent_row<T>(p, row);
}

// A layer whose queries come out of a latent of their own: RMS-normed query latents [rows, q_pad] (zeros behind q_rank), and
// in the same launch the rows' cache entries.  A wave per row; grid.y: 0 the cache, 1 the queries.
struct QueryLatentParams {
  void* out;
  const void* q;
  const float* weight;
  int64_t q_stride;
  int q_rank, q_pad;
};
template <typename T>
__global__ __launch_bounds__(256) void latent_down_kernel(const LatentCacheParams p, const QueryLatentParams z) {
  using S = typename T::store_t;
  constexpr int X = 16 / sizeof(S), N = 4;  // pieces of X a lane keeps
  const int row = blockIdx.x * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
  if (row >= p.rows) return;
  if (blockIdx.y == 0) {
    write_latent_row<T>(p, row);
    return;
  }
  const S* q = (const S*)z.q + row * z.q_stride;
  S* out = (S*)z.out + (int64_t)row * z.q_pad;
  float ss = 0.f;
  if (z.q_rank % X == 0 && z.q_rank <= 64 * X * N && ((uintptr_t)q & 15) == 0) {
    float v[N][X];
#pragma unroll
    for (int i = 0; i < N; ++i) {
      const int d = (i * 64 + lane) * X;
      if (d >= z.q_rank) continue;
      const Vec16<T> raw = *reinterpret_cast<const Vec16<T>*>(q + d);
#pragma unroll
      for (int j = 0; j < X; ++j) {
        v[i][j] = T::to_float(raw.v[j]);
        ss = fmaf(v[i][j], v[i][j], ss);
      }
    }
    const float f = 1.f / sqrtf(wave_sum(ss) / (float)z.q_rank + p.eps);
#pragma unroll
    for (int i = 0; i < N; ++i) {
      const int d = (i * 64 + lane) * X;
      if (d >= z.q_rank) continue;
      Vec16<T> y;
#pragma unroll
      for (int j = 0; j < X; ++j) y.v[j] = T::from_float(v[i][j] * f * z.weight[d + j]);
      *reinterpret_cast<Vec16<T>*>(out + d) = y;
    }
    for (int d = z.q_rank + lane; d < z.q_pad; d += 64) out[d] = T::from_float(0.f);
    return;
  }
  for (int d = lane; d < z.q_rank; d += 64) {
    const float v = T::to_float(q[d]);
    ss = fmaf(v, v, ss);
  }
  const float f = 1.f / sqrtf(wave_sum(ss) / (float)z.q_rank + p.eps);
  for (int d = lane; d < z.q_pad; d += 64) out[d] = T::from_float(d < z.q_rank ? T::to_float(q[d]) * f * z.weight[d] : 0.f);
}

// Rows of a 16-row tile that all belong to one long portion need nothing in latent space.
__device__ __forceinline__ bool tile_is_expanded(const int32_t* qsl, int num_seqs, int row0, int row1, int absorbed_max) {
  const int a = find_seq(qsl, num_seqs, row0);
  return a < num_seqs && qsl[a + 1] > row1 && qsl[a + 1] - qsl[a] > absorbed_max;
}

struct HeadProjectParams {
  void* y;                 // row r, head h, entry n at y + r * y_stride + h * y_head + n
  const void *x, *w, *gate;  // x likewise; w [heads, npad, kpad] (npad a multiple of 16, zero-padded)
  int64_t y_stride, x_stride, gate_stride;
  int y_head, x_head, n, k, npad, kpad, rows, heads;
  const int32_t* query_start_loc;
  int num_seqs, absorbed_max;
  // the tail of a query row: its rotated part at entry n .. n + tail - 1 of y, from x's entries k .. k + rot_dim - 1
  int tail, rot_dim, rot_dims;
  float grow;
  const int64_t* positions;
  const double* turns;
  LatentCacheParams cache;  // the rows' own latents, written by the launch that takes their queries to latent space
};

template <typename T>
__device__ __forceinline__ float project_gate(const HeadProjectParams& p, int row, int head) {
  if (p.gate == nullptr) return 1.f;
  return 1.f / (1.f + expf(-T::to_float(((const typename T::store_t*)p.gate)[row * p.gate_stride + head])));
}

template <typename T>
__device__ __forceinline__ void project_tail(const HeadProjectParams& p, int row0, int head) {
  using S = typename T::store_t;
  const int pairs = p.tail >> 1;
  for (int i = threadIdx.x; i < 16 * pairs; i += 256) {
    const int row = row0 + i / pairs, e = 2 * (i % pairs);
    if (row >= p.rows) break;
    const S* z = (const S*)p.x + row * p.x_stride + (int64_t)head * p.x_head + p.k;
    float u = e < p.rot_dim ? T::to_float(z[e]) : 0.f, v = e + 1 < p.rot_dim ? T::to_float(z[e + 1]) : 0.f;
    if (e < p.rot_dims) {
      float c, s;
      rotation_of(p.positions[row], p.turns[e >> 1], p.grow, c, s);
      const float t = u * c - v * s;
      v = v * c + u * s;
      u = t;
    }
    S* y = (S*)p.y + row * p.y_stride + (int64_t)head * p.y_head + p.n + e;
    y[0] = T::from_float(u);
    y[1] = T::from_float(v);
  }
}

// What a workgroup does besides products; true: nothing else is left to do.
template <typename T>
__device__ __forceinline__ bool beside_products(const HeadProjectParams& p, int row0, int head) {
  const bool last = p.tail > 0 && blockIdx.x == gridDim.x - 1;
  if (last && p.cache.kv != nullptr)  // (the tile's rows are dealt to the heads' workgroups)
    for (int i = 4 * head + (threadIdx.x >> 6); i < 16 && row0 + i < p.rows; i += 4 * p.heads) write_latent_row<T>(p.cache, row0 + i);
  if (p.query_start_loc != nullptr &&
      tile_is_expanded(p.query_start_loc, p.num_seqs, row0, min(row0 + 15, p.rows - 1), p.absorbed_max))
    return true;
  if (last) project_tail<T>(p, row0, head);
  return last;
}

// y[r, h, :] = W_h x[r, h, :] (* sigmoid(gate[r, h])).  grid (n tiles (+ 1 for the tail), heads, 16-row tiles)
template <typename T>
__global__ __launch_bounds__(256) void head_project_simple_kernel(const HeadProjectParams p) {
  using S = typename T::store_t;
  const int head = blockIdx.y, row0 = blockIdx.z * 16;
  if (beside_products<T>(p, row0, head)) return;
  const int row = row0 + (threadIdx.x >> 4), n = blockIdx.x * 16 + (threadIdx.x & 15);
  if (row >= p.rows || n >= p.n) return;
  const S* x = (const S*)p.x + row * p.x_stride + (int64_t)head * p.x_head;
  const S* w = (const S*)p.w + ((int64_t)head * p.npad + n) * p.kpad;
  float acc = 0.f;
  for (int k = 0; k < p.k; ++k) acc = fmaf(T::to_float(x[k]), T::to_float(w[k]), acc);
  ((S*)p.y)[row * p.y_stride + (int64_t)head * p.y_head + n] = T::from_float(acc * project_gate<T>(p, row, head));
}

// The same on 16x16x32 MFMAs: W rows are the A operand, the 16 rows' x the B operand; a wave per 16 outputs.
__global__ __launch_bounds__(256) void head_project_mfma_kernel(const HeadProjectParams p) {
  const int head = blockIdx.y, row0 = blockIdx.z * 16;
  if (beside_products<BF16>(p, row0, head)) return;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, g = lane >> 4, c = lane & 15;
  const int n0 = (blockIdx.x * 4 + wave) * 16;
  if (n0 >= p.npad) return;
  const int row = min(row0 + c, p.rows - 1);
  const uint16_t* x = (const uint16_t*)p.x + row * p.x_stride + (int64_t)head * p.x_head + 8 * g;
  const uint16_t* w = (const uint16_t*)p.w + ((int64_t)head * p.npad + n0 + c) * p.kpad + 8 * g;
  l_f32x4_t acc{0.f, 0.f, 0.f, 0.f};
  constexpr int B = 4;  // k-steps in flight
  for (int k0 = 0; k0 < p.kpad; k0 += 32 * B) {
    uint4 a[B], b[B];
#pragma unroll
    for (int j = 0; j < B; ++j) {
      const int k = k0 + 32 * j;
      a[j] = b[j] = uint4{0, 0, 0, 0};
      if (k < p.kpad) a[j] = *reinterpret_cast<const uint4*>(w + k);
      if (k + 8 * g < p.k) b[j] = *reinterpret_cast<const uint4*>(x + k);
    }
#pragma unroll
    for (int j = 0; j < B; ++j)
      acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(l_bf16x8_t, a[j]), __builtin_bit_cast(l_bf16x8_t, b[j]),
                                                    acc, 0, 0, 0);
  }
  if (row0 + c >= p.rows) return;
  const float f = project_gate<BF16>(p, row, head);
  uint16_t* y = (uint16_t*)p.y + row * p.y_stride + (int64_t)head * p.y_head;
#pragma unroll
  for (int r = 0; r < 4; ++r)
    if (n0 + 4 * g + r < p.n) y[n0 + 4 * g + r] = BF16::from_float(acc[r] * f);
}

static int head_project(const HeadProjectParams& p, int dtype, hipStream_t s) {
  if (p.rows == 0) return 0;
  LV_CHECK(p.heads > 0 && p.heads <= 65535 && p.rows <= 65535 * 16, "too many heads or rows");
  const unsigned tail = p.tail > 0, rt = (p.rows + 15) / 16;
  // 16-byte pieces of x: everything that separates them is a multiple of 8
  const bool vec = ((p.x_stride | p.x_head | p.k) & 7) == 0 && ((uintptr_t)p.x & 15) == 0 && (p.kpad & 31) == 0;
  if (dtype == LVLLM_BF16 && vec) {
    hipLaunchKernelGGL(head_project_mfma_kernel, dim3((p.npad + 63) / 64 + tail, p.heads, rt), dim3(256), 0, s, p);
  } else {
    LV_DISPATCH_F32_BF16(dtype, {
      hipLaunchKernelGGL((head_project_simple_kernel<scalar_t>), dim3((p.n + 15) / 16 + tail, p.heads, rt), dim3(256), 0, s, p);
    });
  }
  LV_LAUNCH_CHECK();
  return 0;
}

// The plain body, for 32-bit elements and sizes without an MFMA instantiation: a workgroup per (row, head), 256 keys a round.
// Its result, [rows, heads, cpad], is the weighted sum in latent space.
template <typename T>
__global__ __launch_bounds__(256) void latent_attention_simple_kernel(const LatentAttnParams p, void* o_lat) {
  using S = typename T::store_t;
  constexpr int x = 16 / sizeof(S);
  extern __shared__ float sm[];
  const int rw = p.cpad + p.rpad;
  float* sq = sm;           // [rw]
  float* sp = sq + rw;      // [256]
  float* sacc = sp + 256;   // [cpad]
  __shared__ float red[16];
  const int row = blockIdx.x, head = blockIdx.y;
  const int seq = find_seq(p.query_start_loc, p.num_seqs, row);
  if (seq >= p.num_seqs) {  // padding rows: whatever is read afterwards is finite
    for (int d = threadIdx.x; d < p.cpad; d += 256) ((S*)o_lat)[((int64_t)row * p.heads + head) * p.cpad + d] = T::from_float(0.f);
    return;
  }
  const int qbeg = p.query_start_loc[seq], qlen = p.query_start_loc[seq + 1] - qbeg;
  if (qlen > p.absorbed_max) return;
  const int pos = p.seq_lens[seq] - qlen + (row - qbeg);
  S* out = (S*)o_lat + ((int64_t)row * p.heads + head) * p.cpad;
  if (pos < 0) {  // a padding row of a captured step
    for (int d = threadIdx.x; d < p.cpad; d += 256) out[d] = T::from_float(0.f);
    return;
  }
  const int lo = first_key(pos, p.window);
  const int32_t* table = p.block_tables + (int64_t)seq * p.max_blocks;
  const S* q = (const S*)p.q + ((int64_t)row * p.heads + head) * rw;
  for (int d = threadIdx.x; d < rw; d += 256) sq[d] = T::to_float(q[d]);
  for (int d = threadIdx.x; d < p.cpad; d += 256) sacc[d] = 0.f;
  const int bs = p.block_size;
  auto row_of = [&](int key) {
    const int b = min(max(table[min(key / bs, p.max_blocks - 1)], 0), p.max_block);
    return (const S*)p.cache + b * p.block_stride + (int64_t)(key % bs) * rw;
  };
  float m = -FLT_MAX, l = 0.f;
  for (int k0 = lo; k0 <= pos; k0 += 256) {
    __syncthreads();
    const int key = k0 + threadIdx.x;
    float score = -FLT_MAX;
    if (key <= pos) {
      const S* kc = row_of(key);
      float acc = 0.f;
      for (int d = 0; d < rw; d += x) {
        const Vec16<T> kv = *reinterpret_cast<const Vec16<T>*>(kc + d);
#pragma unroll
        for (int j = 0; j < x; ++j) acc = fmaf(sq[d + j], T::to_float(kv.v[j]), acc);
      }
      score = acc * p.scale;
    }
    float mx = wave_max(score);
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = mx;
    __syncthreads();
    const float m_new = fmaxf(m, fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3])));
    const float corr = expf(m - m_new);
    const float e = key <= pos ? expf(score - m_new) : 0.f;
    sp[threadIdx.x] = e;
    __syncthreads();
    l = l * corr + block_sum(e, red);
    m = m_new;
    const int nk = min(256, pos + 1 - k0);
    for (int d = threadIdx.x; d < p.cpad; d += 256) {
      float acc = sacc[d] * corr;
      for (int j = 0; j < nk; ++j) acc = fmaf(sp[j], T::to_float(row_of(k0 + j)[d]), acc);
      sacc[d] = acc;
    }
  }
  float f = 1.f / l;
  if (p.sink != nullptr) {
    const float sink = p.sink[head], top = fmaxf(m, sink), own = expf(m - top);
    f = own / (l * own + expf(sink - top));
  }
  for (int d = threadIdx.x; d < p.cpad; d += 256) out[d] = T::from_float(sacc[d] * f);
}

// Rows first[s] .. of every long sequence, back to back (padded to 16 rows a sequence): out[starts[s] + i] = key first[s] + i.
// A wave per row, 16 bytes a lane and turn.
__global__ __launch_bounds__(256) void latent_gather_kernel(char* __restrict__ out, const char* __restrict__ cache,
                                                            const int64_t block_bytes, const int block_size, const int max_block,
                                                            const int row_bytes, const int32_t* __restrict__ starts,
                                                            const int32_t* __restrict__ first,
                                                            const int32_t* __restrict__ seq_lens,
                                                            const int32_t* __restrict__ block_tables, const int max_blocks,
                                                            const int num_seqs, const int n) {
  const int i = blockIdx.x * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
  if (i >= n) return;
  const int seq = find_seq(starts, num_seqs, i);
  char* dst = out + (int64_t)i * row_bytes;
  const int key = seq < num_seqs ? first[seq] + (i - starts[seq]) : -1;
  if (key < 0 || key >= seq_lens[seq]) {  // padding up to the next multiple of 16
    for (int b = lane * 16; b < row_bytes; b += 1024) *reinterpret_cast<uint4*>(dst + b) = uint4{0, 0, 0, 0};
    return;
  }
  const int blk = min(max(block_tables[(int64_t)seq * max_blocks + min(key / block_size, max_blocks - 1)], 0), max_block);
  const char* src = cache + blk * block_bytes + (int64_t)(key % block_size) * row_bytes;
  for (int b = lane * 16; b < row_bytes; b += 1024) *reinterpret_cast<uint4*>(dst + b) = *reinterpret_cast<const uint4*>(src + b);
}

// Gathered rows and their expanded keys / values [n, heads * dim | heads * vdim] -> pages of head_attention's caches:
//   keys [n / 16][heads][kpad / 8][16][8] = [U c | k_rot | 0], values [n / 16][heads][vpad][16].
// A workgroup per (page, head).
__global__ __launch_bounds__(256) void latent_expand_kernel(uint16_t* __restrict__ kc, uint16_t* __restrict__ vc,
                                                            const uint16_t* __restrict__ kv, const int64_t kv_stride,
                                                            const uint16_t* __restrict__ rows, const int row_elems,
                                                            const int cpad, const int heads, const int dim, const int rot_dim,
                                                            const int vdim, const int kpad, const int vpad) {
  extern __shared__ uint16_t sv[];  // [16][vpad + 2]
  const int page = blockIdx.x, head = blockIdx.y;
  uint16_t* k = kc + ((int64_t)page * heads + head) * kpad * 16;
  uint16_t* v = vc + ((int64_t)page * heads + head) * vpad * 16;
  const int64_t r0 = (int64_t)page * 16;
  const bool vec = ((dim | rot_dim | (int)(kv_stride & 7)) & 7) == 0;
  if (vec) {
    for (int i = threadIdx.x; i < kpad * 2; i += 256) {  // chunk i: entries 8 (i / 16) .. of row i % 16
      const int d = i / 16 * 8;
      const int64_t r = r0 + i % 16;
      uint4 t{0, 0, 0, 0};
      if (d < dim) t = *reinterpret_cast<const uint4*>(kv + r * kv_stride + (int64_t)head * dim + d);
      else if (d < dim + rot_dim) t = *reinterpret_cast<const uint4*>(rows + r * row_elems + cpad + d - dim);
      *reinterpret_cast<uint4*>(k + (int64_t)i * 8) = t;
    }
  } else {
    for (int i = threadIdx.x; i < kpad * 16; i += 256) {
      const int d = i / 128 * 8 + i % 8;
      const int64_t r = r0 + i % 128 / 8;
      k[i] = d < dim ? kv[r * kv_stride + (int64_t)head * dim + d]
                     : d < dim + rot_dim ? rows[r * row_elems + cpad + d - dim] : (uint16_t)0;
    }
  }
  const int ld = vpad + 2;
  const uint16_t* src = kv + (int64_t)heads * dim + (int64_t)head * vdim;
  for (int i = threadIdx.x; i < 16 * vpad; i += 256) {
    const int t = i / vpad, d = i - t * vpad;
    sv[t * ld + d] = d < vdim ? src[(r0 + t) * kv_stride + d] : (uint16_t)0;
  }
  __syncthreads();
  for (int i = threadIdx.x; i < vpad * 2; i += 256) {  // 8 tokens of one value entry
    const int d = i >> 1, t0 = (i & 1) * 8;
    uint32_t w[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) w[j] = (uint32_t)sv[(t0 + 2 * j) * ld + d] | ((uint32_t)sv[(t0 + 2 * j + 1) * ld + d] << 16);
    *reinterpret_cast<uint4*>(v + (int64_t)i * 8) = uint4{w[0], w[1], w[2], w[3]};
  }
}

// Queries of long portions as head_attention takes them: [rows, heads, kpad] = [q | rotated | 0].  A thread takes E entries.
template <typename T, int E>
__global__ __launch_bounds__(256) void latent_rotate_query_kernel(typename T::store_t* __restrict__ out,
                                                                  const typename T::store_t* __restrict__ q,
                                                                  const int64_t q_stride, const int heads, const int dim,
                                                                  const int rot_dim, const int kpad,
                                                                  const int64_t* __restrict__ positions,
                                                                  const double* __restrict__ turns, const int rot_dims,
                                                                  const float grow) {
  using S = typename T::store_t;
  struct alignas(E * sizeof(S)) Piece { S v[E]; };
  extern __shared__ float cs[];  // [rot_dims / 2][2]
  const int row = blockIdx.x;
  for (int i = threadIdx.x; i < rot_dims / 2; i += 256) rotation_of(positions[row], turns[i], grow, cs[2 * i], cs[2 * i + 1]);
  __syncthreads();
  const S* x = q + row * q_stride;
  S* y = out + (int64_t)row * heads * kpad;
  const int qd = dim + rot_dim, per = kpad / E;
  for (int i = threadIdx.x; i < heads * per; i += 256) {
    const int h = i / per, d = (i - h * per) * E;
    const S* xh = x + (int64_t)h * qd;
    Piece t;
    if constexpr (E == 1) {
      float v = d < qd ? T::to_float(xh[d]) : 0.f;
      const int r = d - dim;
      if (r >= 0 && r < rot_dims) {
        const float w = T::to_float(xh[dim + (r ^ 1)]), c = cs[r & ~1], s = cs[r | 1];
        v = r & 1 ? v * c + w * s : v * c - w * s;
      }
      t.v[0] = T::from_float(v);
    } else {  // (dim, rot_dim and rot_dims are multiples of E)
      if (d < qd) {
        t = *reinterpret_cast<const Piece*>(xh + d);
        const int r = d - dim;
        if (r >= 0 && r < rot_dims) {
#pragma unroll
          for (int e = 0; e < E; e += 2) {
            const float u = T::to_float(t.v[e]), v = T::to_float(t.v[e + 1]), c = cs[r + e], s = cs[r + e + 1];
            t.v[e] = T::from_float(u * c - v * s);
            t.v[e + 1] = T::from_float(v * c + u * s);
          }
        }
      } else {
#pragma unroll
        for (int e = 0; e < E; ++e) t.v[e] = T::from_float(0.f);
      }
    }
    *reinterpret_cast<Piece*>(y + (int64_t)i * E) = t;
  }
}

}  // namespace lvllm

using namespace lvllm;

static int cache_params(LatentCacheParams& p, void* cache, int64_t block_stride, int64_t num_blocks, int block_size, int cpad,
                        int rpad, const void* kv, int64_t kv_stride, int kv_rank, int rot_dim, const float* weight, float eps,
                        const int64_t* positions, const double* turns, int rot_dims, float grow, const int64_t* slot_mapping,
                        int rows) {
  LV_CHECK(num_blocks * block_size < ((int64_t)1 << 32), "too many slots");
  LV_CHECK(kv_rank > 0 && kv_rank <= cpad && cpad % 8 == 0 && rot_dim >= 0 && rot_dim <= rpad && rpad % 8 == 0 &&
               rot_dims <= rot_dim && rot_dims % 2 == 0, "latent sizes");
  p.cache = cache; p.block_stride = block_stride; p.num_slots = num_blocks * block_size; p.block_size = block_size;
  p.cpad = cpad; p.rpad = rpad; p.kv = kv; p.kv_stride = kv_stride; p.kv_rank = kv_rank; p.rot_dim = rot_dim;
  p.weight = weight; p.eps = eps; p.positions = positions; p.turns = turns; p.rot_dims = rot_dims;
  p.grow = grow; p.slot_mapping = slot_mapping; p.rows = rows;
  return 0;
}

extern "C" int lvllm_latent_cache(void* cache, int64_t block_stride, int64_t num_blocks, int block_size, int cpad, int rpad,
                                  const void* kv, int64_t kv_stride, int kv_rank, int rot_dim, const float* weight, float eps,
                                  const int64_t* positions, const double* turns, int rot_dims, float grow,
                                  const int64_t* slot_mapping, int rows, int dtype, void* stream) {
  if (rows == 0) return 0;
  LatentCacheParams p{};
  if (int rc = cache_params(p, cache, block_stride, num_blocks, block_size, cpad, rpad, kv, kv_stride, kv_rank, rot_dim, weight,
                            eps, positions, turns, rot_dims, grow, slot_mapping, rows)) return rc;
  LV_DISPATCH_F32_BF16(dtype, {
    hipLaunchKernelGGL((latent_cache_kernel<scalar_t>), dim3((rows + 3) / 4), dim3(256), 0, (hipStream_t)stream, p);
  });
  LV_LAUNCH_CHECK();
  return 0;
}

extern "C" int lvllm_latent_down(void* out, const void* q, int64_t q_stride, int q_rank, int q_pad, const float* q_weight,
                                 void* cache, int64_t block_stride, int64_t num_blocks, int block_size, int cpad, int rpad,
                                 const void* kv, int64_t kv_stride, int kv_rank, int rot_dim, const float* weight, float eps,
                                 const int64_t* positions, const double* turns, int rot_dims, float grow,
                                 const int64_t* slot_mapping, int rows, int dtype, void* stream) {
  if (rows == 0) return 0;
  LV_CHECK(q_rank > 0 && q_rank <= q_pad && q_pad % 8 == 0, "query latents of zero or of more than the padded size");
  LatentCacheParams p{};
  if (int rc = cache_params(p, cache, block_stride, num_blocks, block_size, cpad, rpad, kv, kv_stride, kv_rank, rot_dim, weight,
                            eps, positions, turns, rot_dims, grow, slot_mapping, rows)) return rc;
  const QueryLatentParams z{out, q, q_weight, q_stride, q_rank, q_pad};
  LV_DISPATCH_F32_BF16(dtype, {
    hipLaunchKernelGGL((latent_down_kernel<scalar_t>), dim3((rows + 3) / 4, 2), dim3(256), 0, (hipStream_t)stream, p, z);
  });
  LV_LAUNCH_CHECK();
  return 0;
}

extern "C" int lvllm_latent_query(void* out, const void* q, int64_t q_stride, const void* uk_t, int heads, int dim, int dpad,
                                  int cpad, int rpad, int rot_dim, int rot_dims, const int64_t* positions,
                                  const double* turns, float grow, const int32_t* query_start_loc, int num_seqs,
                                  int absorbed_max, void* cache, int64_t block_stride, int64_t num_blocks, int block_size,
                                  const void* kv, int64_t kv_stride, int kv_rank, const float* weight, float eps,
                                  const int64_t* slot_mapping, int rows, int dtype, void* stream) {
  LV_CHECK(dim > 0 && dim <= dpad && rot_dim <= rpad && rot_dims <= rot_dim && rot_dims % 2 == 0 && cpad % 16 == 0 &&
               rpad > 0 && rpad % 2 == 0, "latent sizes");
  HeadProjectParams p{};
  p.y = out; p.y_stride = (int64_t)heads * (cpad + rpad); p.y_head = cpad + rpad; p.n = cpad; p.npad = cpad;
  p.x = q; p.x_stride = q_stride; p.x_head = dim + rot_dim; p.k = dim; p.kpad = dpad; p.w = uk_t;
  p.rows = rows; p.heads = heads; p.num_seqs = num_seqs; p.absorbed_max = absorbed_max;
  p.query_start_loc = absorbed_max < rows ? query_start_loc : nullptr;  // (no portion can be longer)
  p.tail = rpad; p.rot_dim = rot_dim; p.rot_dims = rot_dims; p.grow = grow; p.positions = positions;
  p.turns = turns;
  if (kv != nullptr)
    if (int rc = cache_params(p.cache, cache, block_stride, num_blocks, block_size, cpad, rpad, kv, kv_stride, kv_rank, rot_dim,
                              weight, eps, positions, turns, rot_dims, grow, slot_mapping, rows)) return rc;
  return head_project(p, dtype, (hipStream_t)stream);
}

// Shares the keys of a sequence are cut into: a workgroup per CU (two where their tiles fit its LDS), none of under 128 keys
static int latent_shares(int rows, int num_seqs, int heads, int cpad, int rpad, int max_query_len, int max_keys) {
  const int64_t cols = (int64_t)heads * max_query_len;
  const int64_t wgs = num_seqs * (cols <= 16 ? 1 : (cols + 31) / 32);
  const int64_t room = 2 * 128 * (cpad + rpad) * 2 <= 150 * 1024 ? 512 : 256;
  int64_t n = (room + wgs - 1) / wgs;
  const int64_t most = (max_keys + 127) / 128, part = ((int64_t)64 << 20) / ((int64_t)rows * heads) + 1;
  n = n < most ? n : most;
  n = n < part ? n : part;
  return n < 1 ? 1 : n > 64 ? 64 : (int)n;
}

static int latent_max_keys(int max_seq_len, int window, int max_query_len) {
  const int64_t w = (int64_t)window + max_query_len + 16;
  return window > 0 && w < max_seq_len ? (int)w : max_seq_len;
}

extern "C" int64_t lvllm_latent_attention_workspace_bytes(int rows, int num_seqs, int heads, int cpad, int rpad,
                                                          int block_size, int window, int absorbed_max, int max_query_len,
                                                          int max_seq_len, int dtype) {
  if (rows <= 0 || num_seqs <= 0 || heads <= 0) return 0;
  if (!latent_takes_mfma(cpad, rpad, block_size, dtype)) return (int64_t)rows * heads * cpad * (dtype == LVLLM_F32 ? 4 : 2);
  const int q = max_query_len < absorbed_max ? max_query_len : absorbed_max;
  const int n = latent_shares(rows, num_seqs, heads, cpad, rpad, q, latent_max_keys(max_seq_len, window, q));
  return (int64_t)rows * heads * n * (cpad + 2) * 4;
}

extern "C" int lvllm_latent_attention(void* out, int64_t out_stride, const void* q, const void* cache, int64_t block_stride,
                                      int64_t num_blocks, int block_size, int cpad, int rpad, const void* uv, int vdim, int vpad,
                                      const void* gate, int64_t gate_stride, const float* sink,
                                      const int32_t* block_tables, int max_blocks, const int32_t* seq_lens,
                                      const int32_t* query_start_loc, int num_seqs, int rows, int heads, float scale,
                                      int window, int absorbed_max, int max_query_len, int max_seq_len, void* workspace,
                                      int64_t workspace_bytes, int dtype, void* stream) {
  if (rows == 0 || num_seqs == 0) return 0;
  LV_CHECK(heads > 0 && heads <= 65535 && num_seqs <= 65535 && max_query_len > 0, "too many heads or sequences, or no query");
  LV_CHECK(cpad > 0 && cpad % 16 == 0 && rpad % 16 == 0 && cpad <= 8192 && rpad <= 2048, "rows are multiples of 16 elements");
  LV_CHECK(max_blocks > 0 && num_blocks > 0 && block_size > 0, "an empty cache");
  LV_CHECK(vdim > 0 && vdim <= vpad && vpad % 16 == 0, "value sizes");
  LV_CHECK(workspace != nullptr &&
               workspace_bytes >= lvllm_latent_attention_workspace_bytes(rows, num_seqs, heads, cpad, rpad, block_size, window,
                                                                         absorbed_max, max_query_len, max_seq_len, dtype),
           "workspace too small (see lvllm_latent_attention_workspace_bytes)");
  LatentAttnParams p{};
  p.out = out; p.out_stride = out_stride; p.q = q; p.cache = cache; p.block_tables = block_tables; p.seq_lens = seq_lens;
  p.query_start_loc = query_start_loc; p.num_seqs = num_seqs; p.rows = rows; p.heads = heads; p.cpad = cpad; p.rpad = rpad;
  p.max_blocks = max_blocks; p.block_size = block_size; p.max_block = (int)(num_blocks - 1); p.nsplit = 1; p.window = window;
  p.absorbed_max = absorbed_max; p.scale = scale; p.block_stride = block_stride; p.uv = uv; p.vdim = vdim; p.vpad = vpad;
  p.gate = gate; p.gate_stride = gate_stride; p.sink = sink;
  p.max_query_len = max_query_len < absorbed_max ? max_query_len : absorbed_max;
  hipStream_t s = (hipStream_t)stream;
  if (latent_takes_mfma(cpad, rpad, block_size, dtype)) {
    p.nsplit = latent_shares(rows, num_seqs, heads, cpad, rpad, p.max_query_len,
                             latent_max_keys(max_seq_len, window, p.max_query_len));
    p.part_o = (float*)workspace;
    p.part_ml = p.part_o + (int64_t)rows * heads * p.nsplit * cpad;
    return launch_latent_mfma(p, s);
  }
  LV_DISPATCH_F32_BF16(dtype, {
    hipLaunchKernelGGL((latent_attention_simple_kernel<scalar_t>), dim3(rows, heads), dim3(256),
                       (size_t)(2 * cpad + rpad + 256) * 4, s, p, workspace);
  });
  LV_LAUNCH_CHECK();
  HeadProjectParams v{};
  v.y = out; v.y_stride = out_stride; v.y_head = vdim; v.n = vdim; v.npad = vpad;
  v.x = workspace; v.x_stride = (int64_t)heads * cpad; v.x_head = cpad; v.k = cpad; v.kpad = cpad; v.w = uv;
  v.gate = gate; v.gate_stride = gate_stride;
  v.rows = rows; v.heads = heads; v.num_seqs = num_seqs; v.absorbed_max = absorbed_max;
  v.query_start_loc = absorbed_max < rows ? query_start_loc : nullptr;  // (no portion can be longer)
  return head_project(v, dtype, s);
}

extern "C" int lvllm_latent_gather(void* out, const void* cache, int64_t block_stride, int64_t num_blocks, int block_size,
                                   int row_elems, const int32_t* starts, const int32_t* first, const int32_t* seq_lens,
                                   const int32_t* block_tables, int max_blocks, int num_seqs, int n, int dtype, void* stream) {
  if (n == 0) return 0;
  const int es = dtype == LVLLM_F32 ? 4 : 2;
  LV_CHECK(row_elems * es % 16 == 0 && block_stride * es % 16 == 0, "rows of 16-byte pieces");
  hipLaunchKernelGGL(latent_gather_kernel, dim3((n + 3) / 4), dim3(256), 0, (hipStream_t)stream, (char*)out,
                     (const char*)cache, block_stride * es, block_size, (int)(num_blocks - 1), row_elems * es, starts, first,
                     seq_lens, block_tables, max_blocks, num_seqs, n);
  LV_LAUNCH_CHECK();
  return 0;
}

extern "C" int lvllm_latent_expand(void* key_pages, void* value_pages, const void* kv, int64_t kv_stride, const void* rows,
                                   int row_elems, int cpad, int n, int heads, int dim, int rot_dim, int vdim, int kpad,
                                   int vpad, int dtype, void* stream) {
  if (n == 0) return 0;
  LV_CHECK(dtype == LVLLM_BF16 && n % 16 == 0 && kpad % 8 == 0 && dim + rot_dim <= kpad && vdim <= vpad && heads <= 65535 &&
               vpad <= 1024, "bf16 pages of 16 rows");
  hipLaunchKernelGGL(latent_expand_kernel, dim3(n / 16, heads), dim3(256), 16 * (vpad + 2) * 2, (hipStream_t)stream,
                     (uint16_t*)key_pages, (uint16_t*)value_pages, (const uint16_t*)kv, kv_stride, (const uint16_t*)rows,
                     row_elems, cpad, heads, dim, rot_dim, vdim, kpad, vpad);
  LV_LAUNCH_CHECK();
  return 0;
}

extern "C" int lvllm_latent_rotate_query(void* out, const void* q, int64_t q_stride, int heads, int dim, int rot_dim, int kpad,
                                         const int64_t* positions, const double* turns, int rot_dims, float grow, int rows,
                                         int dtype, void* stream) {
  if (rows == 0) return 0;
  LV_CHECK(dim + rot_dim <= kpad && rot_dims <= rot_dim && rot_dims % 2 == 0 && rot_dims <= 4096, "query sizes");
  const int e = dtype == LVLLM_F32 ? 4 : 8;
  const bool vec = ((dim | rot_dim | rot_dims | kpad) % e == 0) && q_stride % e == 0 && ((uintptr_t)q & 15) == 0;
  LV_DISPATCH_F32_BF16(dtype, {
    using S = typename scalar_t::store_t;
    if (vec)
      hipLaunchKernelGGL((latent_rotate_query_kernel<scalar_t, 16 / sizeof(S)>), dim3(rows), dim3(256),
                         (size_t)rot_dims * 4 + 8, (hipStream_t)stream, (S*)out, (const S*)q, q_stride, heads, dim, rot_dim,
                         kpad, positions, turns, rot_dims, grow);
    else
      hipLaunchKernelGGL((latent_rotate_query_kernel<scalar_t, 1>), dim3(rows), dim3(256), (size_t)rot_dims * 4 + 8,
                         (hipStream_t)stream, (S*)out, (const S*)q, q_stride, heads, dim, rot_dim, kpad, positions, turns,
                         rot_dims, grow);
  });
  LV_LAUNCH_CHECK();
  return 0;
}
