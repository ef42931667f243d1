// Linear recurrences with a matrix state per head and one decay per key channel, for gfx950:
//
//     S_t = diag(w_t) S_{t-1} + k_t v_t^T          S [dk, dv], fp32, carried per sequence
//     o_t = S_t^T q_t                              (plain read-out), or
//     o_t = (S_{t-1} + diag(u) k_t v_t^T)^T q_t    (bonus read-out: u weighs the current token)
//
// and the low-rank data-dependent decays that drive them:
//
//     z = A f(u_t) + bias,   ln w = logsigmoid(z) / tau   (f = identity)   or   ln w = -exp(z)   (f = tanh)
//
// Everything but the projections' results (q, k, v, the low-rank input) is fp32: decays and their logarithms, the state,
// the read-out.  Rows are the new tokens of `num_seqs` sequences back to back (query_start_loc); a sequence whose tokens
// are all in this step (seq_lens == its rows) starts from a zero state, every other one from its slot.
#include "common.h"

namespace lvllm {

enum { kDecayLogSigmoid = 0, kDecayNegExp = 1 };

__device__ __forceinline__ float log_decay_of(float z, int kind, float inv_tau) {
  if (kind == kDecayNegExp) return -expf(z);
  return (fminf(z, 0.f) - log1pf(expf(-fabsf(z)))) * inv_tau;
}

// ---- ln w [rows, channels] ---------------------------------------------------------------------------------------
constexpr int kDecayRows = 8;
template <typename T>
__global__ __launch_bounds__(256) void log_decay_kernel(float* __restrict__ out, const typename T::store_t* __restrict__ u,
                                                        const int64_t u_stride, const float* __restrict__ a_t,  // [rank, channels]
                                                        const float* __restrict__ bias, const int kind,
                                                        const float inv_tau, const int rows, const int rank,
                                                        const int channels) {
  extern __shared__ float su[];  // [kDecayRows][rank]
  const int row0 = blockIdx.y * kDecayRows;
  const int nr = min(kDecayRows, rows - row0);
  for (int i = threadIdx.x; i < kDecayRows * rank; i += blockDim.x) {
    const int r = i / rank, c = i - r * rank;
    float f = r < nr ? T::to_float(u[(row0 + r) * u_stride + c]) : 0.f;
    su[i] = kind == kDecayNegExp ? tanhf(f) : f;
  }
  __syncthreads();
  const int ch = blockIdx.x * blockDim.x + threadIdx.x;
  if (ch >= channels) return;
  float acc[kDecayRows];
#pragma unroll
  for (int r = 0; r < kDecayRows; ++r) acc[r] = 0.f;
  for (int c = 0; c < rank; ++c) {
    const float w = a_t[(int64_t)c * channels + ch];
#pragma unroll
    for (int r = 0; r < kDecayRows; ++r) acc[r] = fmaf(su[r * rank + c], w, acc[r]);
  }
  const float b = bias[ch];
#pragma unroll
  for (int r = 0; r < kDecayRows; ++r)
    if (r < nr) out[(int64_t)(row0 + r) * channels + ch] = log_decay_of(acc[r] + b, kind, inv_tau);
}

// ---- token-by-token scan -----------------------------------------------------------------------------------------
// One workgroup per (sequence, head, 64 value columns): wave w holds state rows [w * NR, w * NR + NR) of its 64 columns
// in registers, tokens come in tiles of kScanTile through LDS, the four waves' partial read-outs meet in LDS per tile.
struct ScanParams {
  float* o;                        // [rows, heads, dv]
  const void *q, *k, *v;           // row r, head h at r * stride + h * dk (dv)
  int64_t q_stride, k_stride, v_stride;
  const float* log_decay;          // [rows, heads, dk]
  const float* bonus;              // [heads, dk] or null
  float q_scale;
  float* state;                    // [slots, heads, dk, dv], slots state_stride apart
  int64_t state_stride;
  const int32_t *state_slots, *query_start_loc, *seq_lens;
  int num_slots, heads, dk, dv;
};

constexpr int kScanTile = 16;

template <typename T, int NR>
__global__ __launch_bounds__(256) void scan_kernel(const ScanParams p) {
  using S = typename T::store_t;
  extern __shared__ float sm[];
  constexpr int DK = 4 * NR;
  float* sq = sm;                          // [tile][DK]
  float* sk = sq + kScanTile * DK;         // [tile][DK]
  float* sw = sk + kScanTile * DK;         // [tile][DK]
  float* sv = sw + kScanTile * DK;         // [tile][64]
  float* so = sv + kScanTile * 64;         // [4][tile][64]
  float* sb = so + 4 * kScanTile * 64;     // [DK]
  const int head = blockIdx.x, v0 = blockIdx.y * 64, seq = blockIdx.z;
  const int lane = threadIdx.x & 63;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int qbeg = p.query_start_loc[seq], qlen = p.query_start_loc[seq + 1] - qbeg;
  if (qlen <= 0) return;
  const int slot = p.state_slots[seq];
  const bool live = slot >= 0 && slot < p.num_slots;
  const int col = v0 + lane;
  const bool col_ok = col < p.dv;
  float* st = p.state + (int64_t)(live ? slot : 0) * p.state_stride + (int64_t)head * p.dk * p.dv + col;
  const bool fresh = p.seq_lens[seq] <= qlen || !live;
  float s[NR];
#pragma unroll
  for (int i = 0; i < NR; ++i) {
    const int r = wave * NR + i;
    s[i] = (!fresh && col_ok && r < p.dk) ? st[(int64_t)r * p.dv] : 0.f;
  }
  const bool has_bonus = p.bonus != nullptr;
  for (int i = threadIdx.x; i < DK; i += 256) sb[i] = (has_bonus && i < p.dk) ? p.bonus[head * p.dk + i] : 0.f;

  for (int t0 = 0; t0 < qlen; t0 += kScanTile) {
    const int nt = min(kScanTile, qlen - t0);
    __syncthreads();
    for (int i = threadIdx.x; i < kScanTile * DK; i += 256) {
      const int t = i / DK, d = i - t * DK;
      const bool ok = t < nt && d < p.dk;
      const int64_t row = qbeg + t0 + t;
      sq[i] = ok ? T::to_float(((const S*)p.q)[row * p.q_stride + head * p.dk + d]) * p.q_scale : 0.f;
      sk[i] = ok ? T::to_float(((const S*)p.k)[row * p.k_stride + head * p.dk + d]) : 0.f;
      sw[i] = ok ? expf(p.log_decay[(row * p.heads + head) * p.dk + d]) : 1.f;
    }
    for (int i = threadIdx.x; i < kScanTile * 64; i += 256) {
      const int t = i >> 6, d = v0 + (i & 63);
      sv[i] = (t < nt && d < p.dv) ? T::to_float(((const S*)p.v)[(qbeg + t0 + t) * p.v_stride + head * p.dv + d]) : 0.f;
    }
    __syncthreads();
    for (int t = 0; t < nt; ++t) {
      const float vv = sv[t * 64 + lane];
      const float* q = sq + t * DK + wave * NR;
      const float* k = sk + t * DK + wave * NR;
      const float* w = sw + t * DK + wave * NR;
      float acc = 0.f;
      if (has_bonus) {
        const float* u = sb + wave * NR;
#pragma unroll
        for (int i = 0; i < NR; ++i) {
          const float kv = k[i] * vv;
          acc = fmaf(q[i], fmaf(u[i], kv, s[i]), acc);
          s[i] = fmaf(w[i], s[i], kv);
        }
      } else {
#pragma unroll
        for (int i = 0; i < NR; ++i) {
          s[i] = fmaf(w[i], s[i], k[i] * vv);
          acc = fmaf(q[i], s[i], acc);
        }
      }
      so[(wave * kScanTile + t) * 64 + lane] = acc;
    }
    __syncthreads();
    for (int i = threadIdx.x; i < nt * 64; i += 256) {
      const int t = i >> 6, d = v0 + (i & 63);
      if (d < p.dv) {
        const float r = (so[i] + so[kScanTile * 64 + i]) + (so[2 * kScanTile * 64 + i] + so[3 * kScanTile * 64 + i]);
        p.o[((int64_t)(qbeg + t0 + t) * p.heads + head) * p.dv + d] = r;
      }
    }
  }
  if (live && col_ok) {
#pragma unroll
    for (int i = 0; i < NR; ++i) {
      const int r = wave * NR + i;
      if (r < p.dk) st[(int64_t)r * p.dv] = s[i];
    }
  }
}

template <typename T, int NR>
static int launch_scan(const ScanParams& p, int num_seqs, hipStream_t s) {
  const size_t smem = (size_t)(kScanTile * (3 * 4 * NR + 64 + 4 * 64) + 4 * NR) * sizeof(float);
  if (smem > 64 * 1024)
    (void)hipFuncSetAttribute((const void*)scan_kernel<T, NR>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)smem);
  hipLaunchKernelGGL((scan_kernel<T, NR>), dim3(p.heads, (p.dv + 63) / 64, num_seqs), dim3(256), smem, s, p);
  return 0;
}

}  // namespace lvllm

using namespace lvllm;

extern "C" int lvllm_log_decay(float* out, const void* u, int64_t u_stride, const float* a_t, const float* bias, int kind,
                               float inv_tau, int rows, int rank, int channels, int dtype, void* stream) {
  if (rows == 0) return 0;
  LV_CHECK(kind == kDecayLogSigmoid || kind == kDecayNegExp, "unknown decay kind");
  LV_CHECK(rank > 0 && rank <= 1024 && channels > 0, "rank must be in 1 .. 1024");
  const int ny = (rows + kDecayRows - 1) / kDecayRows;
  LV_CHECK(ny <= 65535, "too many rows");
  LV_DISPATCH_DTYPE(dtype, {
    using S = scalar_t::store_t;
    hipLaunchKernelGGL((log_decay_kernel<scalar_t>), dim3((channels + 255) / 256, ny), dim3(256),
                       (size_t)kDecayRows * rank * 4, (hipStream_t)stream, out, (const S*)u, u_stride, a_t, bias, kind,
                       inv_tau, rows, rank, channels);
  });
  LV_LAUNCH_CHECK();
  return 0;
}

extern "C" int lvllm_recurrent_scan(float* o, const void* q, const void* k, const void* v, int64_t q_stride,
                                    int64_t k_stride, int64_t v_stride, const float* log_decay, const float* bonus,
                                    float q_scale, float* state, int64_t state_stride, const int32_t* state_slots,
                                    int num_slots, const int32_t* query_start_loc, const int32_t* seq_lens, int num_seqs,
                                    int heads, int dk, int dv, int dtype, void* stream) {
  if (num_seqs == 0) return 0;
  LV_CHECK(dk > 0 && dk <= 256 && dv > 0, "key size must be in 1 .. 256");
  LV_CHECK(state_stride >= (int64_t)heads * dk * dv, "state slots overlap");
  const ScanParams p{o, q, k, v, q_stride, k_stride, v_stride, log_decay, bonus, q_scale, state, state_stride,
                     state_slots, query_start_loc, seq_lens, num_slots, heads, dk, dv};
  hipStream_t s = (hipStream_t)stream;
  LV_DISPATCH_DTYPE(dtype, {
    if (dk <= 32) launch_scan<scalar_t, 8>(p, num_seqs, s);
    else if (dk <= 64) launch_scan<scalar_t, 16>(p, num_seqs, s);
    else if (dk <= 128) launch_scan<scalar_t, 32>(p, num_seqs, s);
    else launch_scan<scalar_t, 64>(p, num_seqs, s);
  });
  LV_LAUNCH_CHECK();
  return 0;
}
