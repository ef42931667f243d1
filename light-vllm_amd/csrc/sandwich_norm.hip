// Row-wise operators of decoders that norm what a sublayer reads and what it returns, for gfx950: the embedding with a table of
// token pairs, and one launch between two sublayers:
//   v = y_0 (+ bias_0), or half the sum of two branches' RMS norms, each with its own weight
//   x = x + v * weight / rms(v)
//   h = T(x * next_weight / rms(x))
// Everything is fp32; h, which projections read, is rounded to the element type T once.
//
// A branch comes as rows of T, as the fp32 split-K slabs of a decode GEMM, or as the slots of a mixture of experts, whose rows
// are added.
#include "row_ops.h"

namespace lvllm {

struct SandwichBranch {
  const void* y;          // [rows, width], or with slots [total_slots, width]
  const float* partials;  // when set: [num_partials, rows, width], y is unused
  const int32_t* slots;   // [rows, num_slots] or null
  const float* bias;      // [width] or null
  const float* weight;    // two branches: the weight of this one's norm
  int num_partials, num_slots, total_slots;
};

struct SandwichParams {
  float* x;
  void* h;
  SandwichBranch branch[2];
  const float *weight, *next_weight;
  int rows, width;
  float eps;
};

// A workgroup per row; a thread keeps its ITEMS groups of VEC columns in registers.
template <typename T, int VEC, int ITEMS, int BRANCHES>
__global__ __launch_bounds__(1024) void sandwich_norm_kernel(const SandwichParams p) {
  using S = typename T::store_t;
  constexpr int B = ITEMS <= 2 ? 8 : 4;  // rows in flight
  __shared__ float red[BRANCHES * 16];
  const int row = blockIdx.x;
  const int64_t base = (int64_t)row * p.width;
  auto column = [&](int it) { return (it * (int)blockDim.x + (int)threadIdx.x) * VEC; };
  float v[BRANCHES][ITEMS][VEC], x[ITEMS][VEC];
#pragma unroll
  for (int it = 0; it < ITEMS; ++it) {
#pragma unroll
    for (int j = 0; j < VEC; ++j) x[it][j] = 0.f;
    if (column(it) < p.width) load_vec<F32, VEC>(p.x + base + column(it), x[it]);
  }
#pragma unroll
  for (int b = 0; b < BRANCHES; ++b) {
    const SandwichBranch& r = p.branch[b];
#pragma unroll
    for (int it = 0; it < ITEMS; ++it) {
      const bool ok = column(it) < p.width;
#pragma unroll
      for (int j = 0; j < VEC; ++j) v[b][it][j] = 0.f;
      if (ok && r.bias != nullptr) load_vec<F32, VEC>(r.bias + column(it), v[b][it]);
    }
    auto add_rows = [&](int n, auto load) __attribute__((always_inline)) {
      for (int i0 = 0; i0 < n; i0 += B) {
#pragma unroll
        for (int it = 0; it < ITEMS; ++it) {
          if (column(it) >= p.width) continue;
          float t[B][VEC];
#pragma unroll
          for (int i = 0; i < B; ++i)
            if (i0 + i < n) load(i0 + i, column(it), t[i]);
#pragma unroll
          for (int i = 0; i < B; ++i)
            if (i0 + i < n) {
#pragma unroll
              for (int j = 0; j < VEC; ++j) v[b][it][j] += t[i][j];
            }
        }
      }
    };
    if (r.slots != nullptr) {
      const int32_t* slots = r.slots + (int64_t)row * r.num_slots;
      add_rows(r.num_slots, [&](int i, int c, float (&t)[VEC]) {
        load_vec<T, VEC>((const S*)r.y + (int64_t)min(max(slots[i], 0), r.total_slots - 1) * p.width + c, t);
      });
    } else if (r.partials != nullptr) {
      add_rows(r.num_partials, [&](int i, int c, float (&t)[VEC]) {
        load_vec<F32, VEC>(r.partials + (int64_t)i * p.rows * p.width + base + c, t);
      });
    } else {
      add_rows(1, [&](int, int c, float (&t)[VEC]) { load_vec<T, VEC>((const S*)r.y + base + c, t); });
    }
  }
  auto squares = [&](const float (&a)[ITEMS][VEC]) {
    float ss = 0.f;
#pragma unroll
    for (int it = 0; it < ITEMS; ++it)
#pragma unroll
      for (int j = 0; j < VEC; ++j) ss = fmaf(a[it][j], a[it][j], ss);
    return ss;
  };
  auto inv_rms = [&](float ss) { return 1.f / sqrtf(ss / (float)p.width + p.eps); };
  if constexpr (BRANCHES == 2) {
    const float2 ss = block_sum2(squares(v[0]), squares(v[1]), red);
    const float f0 = 0.5f * inv_rms(ss.x), f1 = 0.5f * inv_rms(ss.y);
#pragma unroll
    for (int it = 0; it < ITEMS; ++it) {
      if (column(it) >= p.width) continue;
      float w0[VEC], w1[VEC];
      load_vec<F32, VEC>(p.branch[0].weight + column(it), w0);
      load_vec<F32, VEC>(p.branch[1].weight + column(it), w1);
#pragma unroll
      for (int j = 0; j < VEC; ++j) v[0][it][j] = v[0][it][j] * f0 * w0[j] + v[1][it][j] * f1 * w1[j];
    }
  }
  const float f = inv_rms(block_sum(squares(v[0]), red));
#pragma unroll
  for (int it = 0; it < ITEMS; ++it) {
    if (column(it) >= p.width) continue;
    float w[VEC];
    load_vec<F32, VEC>(p.weight + column(it), w);
#pragma unroll
    for (int j = 0; j < VEC; ++j) x[it][j] = fmaf(v[0][it][j] * f, w[j], x[it][j]);
    store_vec<F32, VEC>(p.x + base + column(it), x[it]);
  }
  const float g = inv_rms(block_sum(squares(x), red));
#pragma unroll
  for (int it = 0; it < ITEMS; ++it) {
    if (column(it) >= p.width) continue;
    float w[VEC];
    load_vec<F32, VEC>(p.next_weight + column(it), w);
#pragma unroll
    for (int j = 0; j < VEC; ++j) w[j] *= x[it][j] * g;
    store_vec<T, VEC>((S*)p.h + base + column(it), w);
  }
}

struct PairEmbedParams {
  float* x;
  void* h;
  const void *table, *pairs;  // pairs null: no second table
  const int64_t* ids;
  int32_t* previous;          // [slots]: a sequence's last token
  const int32_t *state_slots, *query_start_loc, *seq_lens;
  const float* weight;        // of the norm in front of the first sublayer
  int64_t mul_previous, mul_current;
  int buckets, num_seqs, num_slots, vocab, width;
  float eps;
};

// x = table[token] + pairs[(previous * mul_previous + token * mul_current) mod buckets] (a sequence's first token: row
// `buckets`), h = T(x * weight / rms(x)).  A workgroup per row.  The workgroup of a portion's FIRST row also stores the
// sequence's last token: it is the one that has read the old one.
template <typename T, int VEC, int ITEMS>
__global__ __launch_bounds__(1024) void pair_embed_kernel(const PairEmbedParams p) {
  using S = typename T::store_t;
  __shared__ float red[16];
  const int row = blockIdx.x;
  auto token = [&](int64_t r) { return min(max(p.ids[r], (int64_t)0), (int64_t)p.vocab - 1); };
  const int64_t id = token(row);
  int64_t pair = p.buckets;
  if (p.pairs != nullptr) {
    const int seq = find_seq(p.query_start_loc, p.num_seqs, row);
    if (seq < p.num_seqs) {
      const int qbeg = p.query_start_loc[seq], qlen = p.query_start_loc[seq + 1] - qbeg;
      int64_t before = row > qbeg ? token(row - 1) : -1;
      if (row == qbeg) {
        const int slot = p.state_slots[seq];
        const bool live = slot >= 0 && slot < p.num_slots;
        if (live && p.seq_lens[seq] > qlen) before = min(max(p.previous[slot], 0), p.vocab - 1);
        __syncthreads();  // (every thread has read it)
        if (live && threadIdx.x == 0) p.previous[slot] = (int32_t)token(qbeg + qlen - 1);
      }
      if (before >= 0) pair = (before * p.mul_previous + id * p.mul_current) % p.buckets;
    }
  }
  const int64_t base = (int64_t)row * p.width;
  auto column = [&](int it) { return (it * (int)blockDim.x + (int)threadIdx.x) * VEC; };
  float v[ITEMS][VEC], ss = 0.f;
#pragma unroll
  for (int it = 0; it < ITEMS; ++it) {
    const int c = column(it);
    if (c >= p.width) continue;
    load_vec<T, VEC>((const S*)p.table + id * p.width + c, v[it]);
    if (p.pairs != nullptr) {
      float t[VEC];
      load_vec<T, VEC>((const S*)p.pairs + pair * p.width + c, t);
#pragma unroll
      for (int j = 0; j < VEC; ++j) v[it][j] += t[j];
    }
    store_vec<F32, VEC>(p.x + base + c, v[it]);
#pragma unroll
    for (int j = 0; j < VEC; ++j) ss = fmaf(v[it][j], v[it][j], ss);
  }
  const float f = 1.f / sqrtf(block_sum(ss, red) / (float)p.width + p.eps);
#pragma unroll
  for (int it = 0; it < ITEMS; ++it) {
    const int c = column(it);
    if (c >= p.width) continue;
    float w[VEC];
    load_vec<F32, VEC>(p.weight + c, w);
#pragma unroll
    for (int j = 0; j < VEC; ++j) w[j] *= v[it][j] * f;
    store_vec<T, VEC>((S*)p.h + base + c, w);
  }
}

}  // namespace lvllm

using namespace lvllm;

extern "C" int lvllm_sandwich_norm(float* x, void* h, const lvllm_sandwich_branch* branches, int num_branches,
                                   const float* weight, const float* next_weight, float eps, int rows, int width, int dtype,
                                   void* stream) {
  if (rows == 0) return 0;
  LV_CHECK(num_branches == 1 || num_branches == 2, "one or two branches");
  SandwichParams p{};
  for (int b = 0; b < num_branches; ++b) {
    const lvllm_sandwich_branch& r = branches[b];
    LV_CHECK(r.y != nullptr || r.partials != nullptr, "no sublayer output");
    LV_CHECK(r.slots == nullptr || (r.y != nullptr && r.total_slots > 0), "slots without their rows");
    LV_CHECK(num_branches == 1 || r.weight != nullptr, "two branches need a norm each");
    p.branch[b] = {r.y, r.partials, r.slots, r.bias, r.weight, r.num_partials, r.num_slots, r.total_slots};
  }
  p.x = x; p.h = h; p.weight = weight; p.next_weight = next_weight; p.rows = rows; p.width = width; p.eps = eps;
  hipStream_t s = (hipStream_t)stream;
  const int threads = threads_of(rows, width % 4 == 0 ? width / 4 : width);
#define LV_GO(VEC_, ITEMS_)                                                                                                 \
  LV_DISPATCH_F32_BF16(dtype, {                                                                                             \
    if (num_branches == 1)                                                                                                  \
      hipLaunchKernelGGL((sandwich_norm_kernel<scalar_t, VEC_, ITEMS_, 1>), dim3(rows), dim3(threads), 0, s, p);            \
    else                                                                                                                    \
      hipLaunchKernelGGL((sandwich_norm_kernel<scalar_t, VEC_, ITEMS_, 2>), dim3(rows), dim3(threads), 0, s, p);            \
  })
  LV_ROWS(width, threads, LV_GO)
#undef LV_GO
  LV_LAUNCH_CHECK();
  return 0;
}

extern "C" int lvllm_pair_embed(float* x, void* h, const void* table, const void* pairs, const int64_t* ids, int32_t* previous,
                                const int32_t* state_slots, int num_slots, const int32_t* query_start_loc,
                                const int32_t* seq_lens, int num_seqs, int64_t mul_previous, int64_t mul_current, int buckets,
                                const float* weight, float eps, int rows, int vocab, int width, int dtype, void* stream) {
  if (rows == 0) return 0;
  LV_CHECK(vocab > 0 && width > 0, "an empty table");
  LV_CHECK(pairs == nullptr || (buckets > 0 && previous != nullptr && mul_previous >= 0 && mul_current >= 0),
           "a table of token pairs needs buckets and the sequences' last tokens");
  PairEmbedParams p{};
  p.x = x; p.h = h; p.table = table; p.pairs = pairs; p.ids = ids; p.previous = previous; p.state_slots = state_slots;
  p.query_start_loc = query_start_loc; p.seq_lens = seq_lens; p.weight = weight; p.mul_previous = mul_previous;
  p.mul_current = mul_current; p.buckets = buckets; p.num_seqs = num_seqs; p.num_slots = num_slots; p.vocab = vocab;
  p.width = width; p.eps = eps;
  hipStream_t s = (hipStream_t)stream;
  const int threads = threads_of(rows, width % 4 == 0 ? width / 4 : width);
#define LV_GO(VEC_, ITEMS_)                                                                                          \
  LV_DISPATCH_F32_BF16(dtype, {                                                                                      \
    hipLaunchKernelGGL((pair_embed_kernel<scalar_t, VEC_, ITEMS_>), dim3(rows), dim3(threads), 0, s, p);             \
  })
  LV_ROWS(width, threads, LV_GO)
#undef LV_GO
  LV_LAUNCH_CHECK();
  return 0;
}
