// Recurrences with low-rank data-dependent decays (recurrent.h): the decays, the token-by-token scan, and the mixers' operator.
#include "low_rank_decay.h"
#include "recurrent.h"

namespace lvllm {

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
  LV_CHECK(kind == kDecayLogSigmoid || kind == kDecayNegExp, "unknown decay kind");
  return launch_log_decay(out, u, u_stride, a_t, bias, kind, inv_tau, nullptr, rows, rank, channels, dtype, (hipStream_t)stream);
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

extern "C" int64_t lvllm_recurrent_mix_workspace_bytes(int rows, int num_seqs, int heads, int dk, int dv, int max_query_len) {
  if (max_query_len <= 1) return 0;
  return ((int64_t)rows * heads * dk + segments_workspace(rows, num_seqs, heads, dk, dv, max_query_len)) * 4;
}

extern "C" int lvllm_recurrent_mix(void* out, int64_t out_stride, const void* q, const void* k, const void* v,
                                   int64_t q_stride, int64_t k_stride, int64_t v_stride, const void* u, int64_t u_stride,
                                   const float* a_t, const float* decay_bias, int rank, int kind, float inv_tau,
                                   const float* bonus, float q_scale, const void* gate, int64_t gate_stride,
                                   const float* norm_weight, int norm_head_stride, float eps, float out_scale, float* state,
                                   int64_t state_stride, const int32_t* state_slots, int num_slots,
                                   const int32_t* query_start_loc, const int32_t* seq_lens, int num_seqs, int rows,
                                   int heads, int dk, int dv, int max_query_len, void* workspace,
                                   int64_t workspace_bytes, int dtype, void* stream) {
  if (num_seqs == 0 || rows == 0) return 0;
  LV_CHECK(dk > 0 && dk <= 256 && dv > 0 && dv <= 1024, "key size must be in 1 .. 256, value size in 1 .. 1024");
  LV_CHECK(kind == kDecayLogSigmoid || kind == kDecayNegExp, "unknown decay kind");
  LV_CHECK(rank > 0 && rank <= 512, "rank must be in 1 .. 512");
  LV_CHECK(state_stride >= (int64_t)heads * dk * dv && ((dv & 3) != 0 || (state_stride & 3) == 0),
           "state slots overlap or are unaligned");
  LV_CHECK(num_seqs <= 65535 && heads <= 65535, "too many sequences or heads");
  MixParams p{};
  p.q = q; p.k = k; p.v = v; p.q_stride = q_stride; p.k_stride = k_stride; p.v_stride = v_stride;
  p.u = u; p.u_stride = u_stride; p.a_t = a_t; p.decay_bias = decay_bias; p.kind = kind; p.rank = rank; p.inv_tau = inv_tau;
  p.bonus = bonus; p.q_scale = q_scale; p.state = state; p.state_stride = state_stride; p.state_slots = state_slots;
  p.query_start_loc = query_start_loc; p.seq_lens = seq_lens; p.num_seqs = num_seqs; p.num_slots = num_slots;
  p.heads = heads; p.dk = dk; p.dv = dv; p.out = out; p.out_stride = out_stride; p.gate = gate; p.gate_stride = gate_stride;
  p.norm_weight = norm_weight; p.norm_head_stride = norm_head_stride; p.eps = eps; p.out_scale = out_scale;
  hipStream_t s = (hipStream_t)stream;
  if (max_query_len <= 1) return launch_single_tokens<false>(p, dtype, s);
  LV_CHECK(dtype == LVLLM_BF16 || dtype == LVLLM_F32, "bfloat16 or float32");
  LV_CHECK(workspace != nullptr &&
               workspace_bytes >= lvllm_recurrent_mix_workspace_bytes(rows, num_seqs, heads, dk, dv, max_query_len),
           "workspace too small (see lvllm_recurrent_mix_workspace_bytes)");
  float* ws = (float*)workspace;
  p.log_decay = ws;
  ws += (int64_t)rows * heads * dk;
  plan_segments(p, ws, rows, max_query_len);
  LV_CHECK((int64_t)num_seqs * p.max_segs <= 65535, "too many sequences or too long portions");
  const int esize = dtype == LVLLM_F32 ? 4 : 2;
  p.vec_in = ((dv | v_stride | gate_stride) & 3) == 0 && (((uintptr_t)v | (uintptr_t)gate) & (4 * esize - 1)) == 0;
  p.vec_out = ((dv | out_stride) & 3) == 0 && ((uintptr_t)out & (4 * esize - 1)) == 0;
  if (int rc = lvllm_log_decay((float*)workspace, u, u_stride, a_t, decay_bias, kind, inv_tau, rows, rank, heads * dk, dtype, stream))
    return rc;
  if (dtype == LVLLM_BF16) launch_mix_sized<BF16, BF16, false>(p, s);
  else launch_mix_sized<F32, F32, false>(p, s);
  LV_LAUNCH_CHECK();
  if (p.o == nullptr) return 0;
  return launch_head_norm_gate<true>(out, out_stride, p.o, gate, gate_stride, norm_weight, norm_head_stride, eps, out_scale, rows,
                               heads, dv, dtype, s);
}

extern "C" int lvllm_head_norm_gate(void* out, int64_t out_stride, const float* o, const void* gate, int64_t gate_stride,
                                    const float* weight, int weight_head_stride, float eps, float scale, int rows,
                                    int heads, int vdim, int dtype, void* stream) {
  return launch_head_norm_gate<true>(out, out_stride, o, gate, gate_stride, weight, weight_head_stride, eps, scale, rows, heads, vdim,
                               dtype, (hipStream_t)stream);
}
