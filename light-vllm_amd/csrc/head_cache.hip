// What goes into a paged cache whose key and value sizes differ (and the queries that will read it), for gfx950: per-head RMS
// norms of queries and keys, or rotary positions with an optional norm over all heads at once.
//
//   key_cache   [num_blocks, kv_heads, kpad / x, block_size, x],  x = 16 / sizeof(T)   (padding zeroed)
//   value_cache [num_blocks, kv_heads, vpad, block_size]                             (padding zeroed)
//   q_out       [rows, heads, kpad]                                                  (padding zeroed)
//
// Norms and angles are fp32; what the attention reads is rounded to T once.
#include "rotation.h"
#include "row_ops.h"

namespace lvllm {

// Per-head RMS norm of queries and keys (weights [dim], shared by the heads) and the write of the normed keys and the
// values into a paged cache whose key and value sizes differ:
//   key_cache   [num_blocks, kv_heads, kpad / x, block_size, x],  x = 16 / sizeof(T), kpad >= dim (rest zeroed)
//   value_cache [num_blocks, kv_heads, vpad, block_size],         vpad >= vdim (rest zeroed)
// q_out [rows, heads, kpad] (padding zeroed).  L lanes per (row, head); the values of few rows ride along as further
// "heads" (with_values), those of many go through value_cache_tile_kernel.
template <typename T, int L, int VEC>
__global__ __launch_bounds__(256) void qk_norm_cache_kernel(
    typename T::store_t* __restrict__ q_out, typename T::store_t* __restrict__ key_cache,
    typename T::store_t* __restrict__ value_cache, const typename T::store_t* __restrict__ q,
    const typename T::store_t* __restrict__ k, const typename T::store_t* __restrict__ v, const int64_t row_stride,
    const float* __restrict__ q_weight, const float* __restrict__ k_weight, const float eps, const int rows, const int heads,
    const int kv_heads, const int dim, const int vdim, const int kpad, const int vpad, const bool with_values,
    const int64_t* __restrict__ slot_mapping, const int64_t num_slots, const int block_size, const int64_t k_block_stride,
    const int64_t v_block_stride) {
  using S = typename T::store_t;
  constexpr int x = 16 / sizeof(S);
  const int lane = threadIdx.x % L;
  const int per_row = heads + (with_values ? 2 : 1) * kv_heads;
  const unsigned item = blockIdx.x * (256 / L) + threadIdx.x / L;
  const int row = (int)(item / (unsigned)per_row), h = (int)(item - (unsigned)row * per_row);
  if (row >= rows) return;
  int64_t block = 0;
  int off = 0;
  if (h >= heads) {
    const int64_t slot = slot_mapping[row];
    if (slot < 0 || slot >= num_slots) return;
    block = slot / block_size;
    off = (int)(slot - block * block_size);
  }
  if (h >= heads + kv_heads) {
    const int g = h - heads - kv_heads;
    const S* src = v + row * row_stride + (int64_t)g * vdim;
    S* dst = value_cache + block * v_block_stride + (int64_t)g * vpad * block_size + off;
    for (int d = lane; d < vpad; d += L) dst[(int64_t)d * block_size] = d < vdim ? src[d] : T::from_float(0.f);
    return;
  }
  const bool is_q = h < heads;
  const S* src = (is_q ? q + (int64_t)h * dim : k + (int64_t)(h - heads) * dim) + row * row_stride;
  const float* wt = is_q ? q_weight : k_weight;
  S* dst = is_q ? q_out + ((int64_t)row * heads + h) * kpad
                : key_cache + block * k_block_stride + (int64_t)(h - heads) * kpad * block_size + (int64_t)off * x;
  float f[VEC];
  float ss = 0.f;
  for (int d = lane * VEC; d < dim; d += L * VEC) {
    load_vec<T, VEC>(src + d, f);
#pragma unroll
    for (int j = 0; j < VEC; ++j) ss += f[j] * f[j];
  }
  const bool one_pass = dim <= L * VEC;  // (the values are still in registers)
  const float r = 1.f / sqrtf(group_sum<L>(ss) / dim + eps);
  for (int d = lane * VEC; d < kpad; d += L * VEC) {
    float o[VEC];
    if (d < dim) {
      if (!one_pass) load_vec<T, VEC>(src + d, f);
#pragma unroll
      for (int j = 0; j < VEC; ++j) o[j] = f[j] * r * wt[d + j];
    } else {
#pragma unroll
      for (int j = 0; j < VEC; ++j) o[j] = 0.f;
    }
    store_vec<T, VEC>(is_q ? dst + d : dst + (int64_t)(d / x) * block_size * x + d % x, o);
  }
}

// Values of many rows: a workgroup takes 64 rows of one kv head through LDS.  Its rows are cut into groups of consecutive
// slots inside one aligned 8-slot window; a thread stores a (d, group) as one piece when the group is full.
constexpr int kValueTile = 64;
template <typename S>
__global__ __launch_bounds__(256) void value_cache_tile_kernel(S* __restrict__ value_cache, const S* __restrict__ v,
                                                               const int64_t row_stride, const int rows, const int vdim,
                                                               const int vpad, const int64_t* __restrict__ slot_mapping,
                                                               const int64_t num_slots, const int block_size,
                                                               const int64_t v_block_stride) {
  struct alignas(16) Eight { S e[8]; };
  constexpr int LD = kValueTile + 2;
  extern __shared__ __attribute__((aligned(16))) char smem[];
  S* tile = reinterpret_cast<S*>(smem);  // [vdim][LD]
  __shared__ int64_t slots[kValueTile];
  __shared__ int groups[kValueTile], num_groups;  // first row | length << 8
  const int row0 = blockIdx.x * kValueTile, head = blockIdx.y, nt = min(kValueTile, rows - row0), tid = threadIdx.x;
  if (tid < kValueTile) {
    int64_t s = tid < nt ? slot_mapping[row0 + tid] : -1;
    if (s >= num_slots) s = -1;
    slots[tid] = s;
    const int64_t prev = (int64_t)__shfl_up((long long)s, 1);
    const bool first = s >= 0 && (tid == 0 || prev < 0 || s != prev + 1 || (s & 7) == 0);
    const uint64_t starts = __ballot(first), used = __ballot(s >= 0);
    if (first) {
      const uint64_t above = tid == 63 ? 0 : (starts | ~used) >> (tid + 1);
      const int len = above ? __builtin_ctzll(above) + 1 : 64 - tid;
      groups[__builtin_popcountll(starts & ((1ull << tid) - 1))] = tid | (len << 8);
    }
    if (tid == 0) num_groups = __builtin_popcountll(starts);
  }
  const S* src = v + (int64_t)row0 * row_stride + (int64_t)head * vdim;
  for (int i = tid; i < nt * vdim; i += 256) {
    const int t = i / vdim, d = i - t * vdim;
    tile[d * LD + t] = src[t * row_stride + d];
  }
  __syncthreads();
  const int ng = num_groups;
  for (int i = tid; i < vpad * ng; i += 256) {
    const int d = i / ng, gr = groups[i - d * ng], t = gr & 0xff, len = gr >> 8;
    const int64_t s = slots[t], b = s / block_size;
    S* dst = value_cache + b * v_block_stride + ((int64_t)head * vpad + d) * block_size + (s - b * block_size);
    Eight e;
#pragma unroll
    for (int j = 0; j < 8; ++j) e.e[j] = (d < vdim && j < len) ? tile[d * LD + t + j] : (S)0;
    if (len == 8) {
      *reinterpret_cast<Eight*>(dst) = e;
    } else {
#pragma unroll
      for (int j = 0; j < 8; ++j)
        if (j < len) dst[j] = e.e[j];
    }
  }
}

struct RotaryCacheParams {
  void *q_out, *key_cache, *value_cache;
  const void *q, *k, *v;                // rows `row_stride` apart; v may be k
  int64_t row_stride;
  const float *q_weight, *k_weight;     // norms over all of a row's queries / keys; null: none
  float eps;
  int rows, heads, kv_heads, maps, dim, mpad, vdim, vpad;  // a head: `maps` vectors of dim, mpad each with the padding
  bool with_values;
  const int64_t *positions, *slot_mapping;
  const double* turns;                  // [rot_dims / 2]
  int rot_dims;
  int64_t num_slots;
  int block_size;
  int64_t k_block_stride, v_block_stride;
};

// A workgroup per row.  Entry i of a vector turns with entry i + rot_dims / 2; a thread owns VEC neighbouring entries and reads
// their partners as well.  The row's angles are shared by its heads through LDS.
template <typename T, int VEC>
__global__ __launch_bounds__(256) void rotary_cache_kernel(const RotaryCacheParams p) {
  using S = typename T::store_t;
  constexpr int x = 16 / sizeof(S);
  extern __shared__ float cs[];  // [rot_dims / 2] cosines, then sines
  __shared__ float red[32];
  const int row = blockIdx.x, half = p.rot_dims / 2;
  const S* q = (const S*)p.q + row * p.row_stride;
  const S* k = (const S*)p.k + row * p.row_stride;
  const int64_t pos = p.positions[row], slot = p.slot_mapping[row];
  for (int i = threadIdx.x; i < half; i += 256) rotation_of(pos, p.turns[i], cs[i], cs[half + i]);
  const int nq = p.heads * p.maps, nk = p.kv_heads * p.maps;
  float fq = 1.f, fk = 1.f;
  if (p.q_weight != nullptr || p.k_weight != nullptr) {
    auto squares = [&](const S* src, int n) __attribute__((always_inline)) {
      float ss = 0.f, f[VEC];
      for (int d = threadIdx.x * VEC; d < n; d += 256 * VEC) {
        load_vec<T, VEC>(src + d, f);
#pragma unroll
        for (int j = 0; j < VEC; ++j) ss = fmaf(f[j], f[j], ss);
      }
      return ss;
    };
    const float2 ss = block_sum2(squares(q, nq * p.dim), squares(k, nk * p.dim), red);
    fq = 1.f / sqrtf(ss.x / (float)(nq * p.dim) + p.eps);
    fk = 1.f / sqrtf(ss.y / (float)(nk * p.dim) + p.eps);
  }
  __syncthreads();
  const bool stored = slot >= 0 && slot < p.num_slots;
  const int64_t block = stored ? slot / p.block_size : 0;
  const int off = (int)(stored ? slot - block * p.block_size : 0);
  const int pieces = p.mpad / VEC;
  for (int i = threadIdx.x; i < (nq + (stored ? nk : 0)) * pieces; i += 256) {
    const int h = i / pieces, d = (i - h * pieces) * VEC;
    const bool is_q = h < nq;
    const int hh = is_q ? h : h - nq;
    const S* src = (is_q ? q : k) + hh * p.dim;
    const float* w = is_q ? p.q_weight : p.k_weight;
    const float f = is_q ? fq : fk;
    float o[VEC];
    if (d < p.dim) {
      load_vec<T, VEC>(src + d, o);
      if (w != nullptr) {
#pragma unroll
        for (int j = 0; j < VEC; ++j) o[j] *= f * w[hh * p.dim + d + j];
      }
      if (d < p.rot_dims) {
        const bool first = d < half;
        const int at = first ? d : d - half, other = first ? d + half : at;
        float t[VEC];
        load_vec<T, VEC>(src + other, t);
        if (w != nullptr) {
#pragma unroll
          for (int j = 0; j < VEC; ++j) t[j] *= f * w[hh * p.dim + other + j];
        }
#pragma unroll
        for (int j = 0; j < VEC; ++j) {
          const float c = cs[at + j], s = cs[half + at + j];
          o[j] = first ? o[j] * c - t[j] * s : o[j] * c + t[j] * s;
        }
      }
    } else {
#pragma unroll
      for (int j = 0; j < VEC; ++j) o[j] = 0.f;
    }
    if (is_q) {
      store_vec<T, VEC>((S*)p.q_out + ((int64_t)row * nq + hh) * p.mpad + d, o);
    } else {
      const int64_t at = block * p.k_block_stride + (int64_t)hh * p.mpad * p.block_size;
      store_vec<T, VEC>((S*)p.key_cache + at + (int64_t)(d / x) * p.block_size * x + off * x + d % x, o);
    }
  }
  if (!p.with_values || !stored) return;
  const S* v = (const S*)p.v + row * p.row_stride;
  for (int i = threadIdx.x; i < p.kv_heads * p.vpad; i += 256) {
    const int g = i / p.vpad, d = i - g * p.vpad;
    S* dst = (S*)p.value_cache + block * p.v_block_stride + ((int64_t)g * p.vpad + d) * p.block_size + off;
    *dst = d < p.vdim ? v[(int64_t)g * p.vdim + d] : T::from_float(0.f);
  }
}

}  // namespace lvllm

using namespace lvllm;

// whether values go through value_cache_tile_kernel, and its LDS
static bool tiled_values(int rows, int vdim, int esize, int block_size, const void* value_cache, int64_t v_block_stride) {
  return rows > 64 && vdim * (kValueTile + 2) * esize <= 64 * 1024 && block_size % 8 == 0 && ((uintptr_t)value_cache & 15) == 0 &&
         v_block_stride * esize % 16 == 0;
}
template <typename S>
static void write_value_tiles(void* value_cache, const void* v, int64_t row_stride, int rows, int kv_heads, int vdim, int vpad,
                              const int64_t* slot_mapping, int64_t num_slots, int block_size, int64_t v_block_stride, hipStream_t s) {
  hipLaunchKernelGGL((value_cache_tile_kernel<S>), dim3((rows + kValueTile - 1) / kValueTile, kv_heads), dim3(256),
                     (size_t)vdim * (kValueTile + 2) * sizeof(S), s, (S*)value_cache, (const S*)v, row_stride, rows, vdim, vpad,
                     slot_mapping, num_slots, block_size, v_block_stride);
}

extern "C" int lvllm_qk_norm_cache(void* q_out, void* key_cache, void* value_cache, const void* q, const void* k,
                                   const void* v, int64_t row_stride, const float* q_weight, const float* k_weight,
                                   float eps, int rows, int heads, int kv_heads, int dim, int vdim, int kpad, int vpad,
                                   const int64_t* slot_mapping, int64_t num_blocks, int block_size,
                                   int64_t k_block_stride, int64_t v_block_stride, int dtype, void* stream) {
  if (rows == 0) return 0;
  LV_CHECK(heads > 0 && kv_heads > 0 && heads % kv_heads == 0, "heads must be a multiple of kv_heads");
  LV_CHECK(dim <= kpad && vdim <= vpad && kpad % 8 == 0, "padded sizes must hold the real ones");
  LV_CHECK(k_block_stride >= (int64_t)kv_heads * kpad * block_size && v_block_stride >= (int64_t)kv_heads * vpad * block_size,
           "cache blocks overlap");
  const int esize = dtype == LVLLM_F32 ? 4 : 2;
  const bool tiled = tiled_values(rows, vdim, esize, block_size, value_cache, v_block_stride);
  const bool vec = ((dim | row_stride) & 3) == 0 && (((uintptr_t)q | (uintptr_t)k) & (4 * esize - 1)) == 0 &&
                   (((uintptr_t)q_out | (uintptr_t)key_cache) & 15) == 0 && k_block_stride * esize % 16 == 0;
  const bool vec8 = vec && esize == 2 && ((dim | row_stride) & 7) == 0 && (((uintptr_t)q | (uintptr_t)k) & 15) == 0;
  const int64_t items = (int64_t)rows * (heads + (tiled ? 1 : 2) * kv_heads);
  LV_CHECK(items <= INT32_MAX && kv_heads <= 65535, "too many rows");
#define LV_QK(VEC_)                                                                                                          \
  hipLaunchKernelGGL((qk_norm_cache_kernel<scalar_t, kL, VEC_>), grid, dim3(256), 0, (hipStream_t)stream, (S*)q_out,          \
                     (S*)key_cache, (S*)value_cache, (const S*)q, (const S*)k, (const S*)v, row_stride, q_weight, k_weight,  \
                     eps, rows, heads, kv_heads, dim, vdim, kpad, vpad, !tiled, slot_mapping, num_blocks * block_size,       \
                     block_size, k_block_stride, v_block_stride)
  LV_DISPATCH_DTYPE(dtype, {
    using S = scalar_t::store_t;
    constexpr int kWide = sizeof(S) == 2 ? 8 : 4;  // elements of a 16-byte piece
    const int lanes = lanes_for(kpad, vec8 ? kWide : vec ? 4 : 1);
    const dim3 grid((unsigned)((items * lanes + 255) / 256));
    LV_LANES(lanes, {
      if (vec8) LV_QK(kWide);
      else if (vec) LV_QK(4);
      else LV_QK(1);
    })
    if (tiled)
      write_value_tiles<S>(value_cache, v, row_stride, rows, kv_heads, vdim, vpad, slot_mapping, num_blocks * block_size,
                           block_size, v_block_stride, (hipStream_t)stream);
  });
#undef LV_QK
  LV_LAUNCH_CHECK();
  return 0;
}

extern "C" int lvllm_rotary_cache(void* q_out, void* key_cache, void* value_cache, const void* q, const void* k, const void* v,
                                  int64_t row_stride, const float* q_weight, const float* k_weight, float eps, int rows,
                                  int heads, int kv_heads, int maps, int dim, int vdim, int kpad, int vpad,
                                  const int64_t* positions, const double* turns, int rot_dims, const int64_t* slot_mapping,
                                  int64_t num_blocks, int block_size, int64_t k_block_stride, int64_t v_block_stride, int dtype,
                                  void* stream) {
  if (rows == 0) return 0;
  LV_CHECK(heads > 0 && kv_heads > 0 && heads % kv_heads == 0, "heads must be a multiple of kv_heads");
  LV_CHECK((maps == 1 || maps == 2) && kpad % (8 * maps) == 0 && dim * maps <= kpad && vdim <= vpad,
           "padded sizes must hold the real ones");
  LV_CHECK(rot_dims >= 0 && rot_dims % 2 == 0 && rot_dims <= dim && rot_dims <= 8192, "rotated entries come in pairs of a head's");
  LV_CHECK(k_block_stride >= (int64_t)kv_heads * kpad * block_size && v_block_stride >= (int64_t)kv_heads * vpad * block_size,
           "cache blocks overlap");
  const int esize = dtype == LVLLM_F32 ? 4 : 2;
  RotaryCacheParams p{};
  p.q_out = q_out; p.key_cache = key_cache; p.value_cache = value_cache; p.q = q; p.k = k; p.v = v; p.row_stride = row_stride;
  p.q_weight = q_weight; p.k_weight = k_weight; p.eps = eps; p.rows = rows; p.heads = heads; p.kv_heads = kv_heads;
  p.maps = maps; p.dim = dim; p.mpad = kpad / maps; p.vdim = vdim; p.vpad = vpad; p.positions = positions;
  p.slot_mapping = slot_mapping; p.turns = turns; p.rot_dims = rot_dims; p.num_slots = num_blocks * block_size;
  p.block_size = block_size; p.k_block_stride = k_block_stride; p.v_block_stride = v_block_stride;
  p.with_values = !tiled_values(rows, vdim, esize, block_size, value_cache, v_block_stride);
  // pieces: of dim, of the rotated half, of the rows, aligned in memory
  const uint64_t sizes = (uint64_t)(dim | (rot_dims / 2) | p.mpad | row_stride);
  const uintptr_t in = (uintptr_t)q | (uintptr_t)k, to = (uintptr_t)q_out | (uintptr_t)key_cache;
  const bool blocks = k_block_stride * esize % 16 == 0 && (to & 15) == 0;
  const bool vec8 = esize == 2 && (sizes & 7) == 0 && (in & 15) == 0 && blocks;
  const bool vec4 = (sizes & 3) == 0 && (in & (4 * esize - 1)) == 0 && blocks;
  hipStream_t s = (hipStream_t)stream;
  LV_DISPATCH_F32_BF16(dtype, {
    using S = typename scalar_t::store_t;
    constexpr int kWide = sizeof(S) == 2 ? 8 : 4;
    const size_t smem = (size_t)rot_dims * sizeof(float);
    if (vec8) hipLaunchKernelGGL((rotary_cache_kernel<scalar_t, kWide>), dim3(rows), dim3(256), smem, s, p);
    else if (vec4) hipLaunchKernelGGL((rotary_cache_kernel<scalar_t, 4>), dim3(rows), dim3(256), smem, s, p);
    else hipLaunchKernelGGL((rotary_cache_kernel<scalar_t, 1>), dim3(rows), dim3(256), smem, s, p);
    if (!p.with_values)
      write_value_tiles<S>(value_cache, v, row_stride, rows, kv_heads, vdim, vpad, slot_mapping, p.num_slots, block_size,
                           v_block_stride, s);
  });
  LV_LAUNCH_CHECK();
  return 0;
}
