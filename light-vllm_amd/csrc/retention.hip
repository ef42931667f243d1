// Retention: the recurrence of recurrent.h with one fixed decay per head, over rotated queries and keys.  Rotated rows are fp32:
// single tokens rotate theirs in the recurrence's launch, chunks read rows that a first launch has rotated.
#include "recurrent.h"

namespace lvllm {

// A workgroup per row: the row's angles once, through LDS; a thread takes VEC neighbouring entries and their partners.
template <typename T, int VEC>
__global__ __launch_bounds__(256) void rotate_rows_kernel(float* __restrict__ q_out, float* __restrict__ k_out,
                                                          const typename T::store_t* __restrict__ q,
                                                          const typename T::store_t* __restrict__ k, const int64_t q_stride,
                                                          const int64_t k_stride, const int64_t* __restrict__ positions,
                                                          const double* __restrict__ turns, const int rot_dims, const int heads,
                                                          const int dk) {
  extern __shared__ float cs[];  // [rot_dims / 2] cosines, then sines
  const int row = blockIdx.x, half = rot_dims / 2, n = heads * dk / VEC;
  for (int i = threadIdx.x; i < half; i += 256) rotation_of(positions[row], turns[i], cs[i], cs[half + i]);
  __syncthreads();
  for (int i = threadIdx.x; i < 2 * n; i += 256) {
    const bool is_q = i < n;
    const int at = (is_q ? i : i - n) * VEC, d = at % dk;
    const typename T::store_t* src = is_q ? q + row * q_stride : k + row * k_stride;
    float v[VEC];
    load_vec<T, VEC>(src + at, v);
    if (d < rot_dims) {
      const bool first = d < half;
      const int pair = first ? d : d - half;
      float t[VEC];
      load_vec<T, VEC>(src + (first ? at + half : at - half), t);
#pragma unroll
      for (int j = 0; j < VEC; ++j) v[j] = v[j] * cs[pair + j] + (first ? -t[j] : t[j]) * cs[half + pair + j];
    }
    store_vec<F32, VEC>((is_q ? q_out : k_out) + (int64_t)row * heads * dk + at, v);
  }
}

}  // namespace lvllm

using namespace lvllm;

extern "C" int64_t lvllm_retention_workspace_bytes(int rows, int num_seqs, int heads, int dk, int dv, int max_query_len) {
  if (max_query_len <= 1) return 0;
  return (2 * (int64_t)rows * heads * dk + segments_workspace(rows, num_seqs, heads, dk, dv, max_query_len)) * 4;
}

extern "C" int lvllm_retention(void* out, int64_t out_stride, const void* q, const void* k, const void* v, int64_t q_stride,
                               int64_t k_stride, int64_t v_stride, const int64_t* positions, const double* turns, int rot_dims,
                               const float* head_decay, float q_scale, const void* gate, int64_t gate_stride,
                               const float* norm_weight, int norm_head_stride, float eps, float out_scale, float* state,
                               int64_t state_stride, const int32_t* state_slots, int num_slots, const int32_t* query_start_loc,
                               const int32_t* seq_lens, int num_seqs, int rows, int heads, int dk, int dv, int max_query_len,
                               void* workspace, int64_t workspace_bytes, int dtype, void* stream) {
  if (num_seqs == 0 || rows == 0) return 0;
  LV_CHECK(dk > 0 && dk <= 256 && dv > 0 && dv <= 1024, "key size must be in 1 .. 256, value size in 1 .. 1024");
  LV_CHECK(rot_dims >= 0 && rot_dims % 2 == 0 && rot_dims <= dk, "rotated entries come in pairs of a head's");
  LV_CHECK(state_stride >= (int64_t)heads * dk * dv && ((dv & 3) != 0 || (state_stride & 3) == 0),
           "state slots overlap or are unaligned");
  LV_CHECK(num_seqs <= 65535 && heads <= 65535, "too many sequences or heads");
  LV_CHECK(dtype == LVLLM_BF16 || dtype == LVLLM_F32, "bfloat16 or float32");
  MixParams p{};
  p.q = q; p.k = k; p.v = v; p.q_stride = q_stride; p.k_stride = k_stride; p.v_stride = v_stride;
  p.head_decay = head_decay; p.positions = positions; p.turns = turns; p.rot_dims = rot_dims;
  p.q_scale = q_scale; p.state = state; p.state_stride = state_stride; p.state_slots = state_slots;
  p.query_start_loc = query_start_loc; p.seq_lens = seq_lens; p.num_seqs = num_seqs; p.num_slots = num_slots;
  p.heads = heads; p.dk = dk; p.dv = dv; p.out = out; p.out_stride = out_stride; p.gate = gate; p.gate_stride = gate_stride;
  p.norm_weight = norm_weight; p.norm_head_stride = norm_head_stride; p.eps = eps; p.out_scale = out_scale;
  hipStream_t s = (hipStream_t)stream;
  if (max_query_len <= 1) return launch_single_tokens<true>(p, dtype, s);
  LV_CHECK(workspace != nullptr &&
               workspace_bytes >= lvllm_retention_workspace_bytes(rows, num_seqs, heads, dk, dv, max_query_len),
           "workspace too small (see lvllm_retention_workspace_bytes)");
  float* ws = (float*)workspace;
  float *qr = ws, *kr = ws + (int64_t)rows * heads * dk;
  plan_segments(p, kr + (int64_t)rows * heads * dk, rows, max_query_len);
  LV_CHECK((int64_t)num_seqs * p.max_segs <= 65535, "too many sequences or too long portions");
  LV_DISPATCH_F32_BF16(dtype, {
    using S = typename scalar_t::store_t;
    const bool vec = ((dk | (rot_dims / 2)) & 3) == 0 && ((q_stride | k_stride) & 3) == 0 &&
                     (((uintptr_t)q | (uintptr_t)k) & (4 * sizeof(S) - 1)) == 0 && ((uintptr_t)qr & 15) == 0;
    const size_t smem = (size_t)rot_dims * sizeof(float);
    if (vec)
      hipLaunchKernelGGL((rotate_rows_kernel<scalar_t, 4>), dim3(rows), dim3(256), smem, s, qr, kr, (const S*)q, (const S*)k,
                         q_stride, k_stride, positions, turns, rot_dims, heads, dk);
    else
      hipLaunchKernelGGL((rotate_rows_kernel<scalar_t, 1>), dim3(rows), dim3(256), smem, s, qr, kr, (const S*)q, (const S*)k,
                         q_stride, k_stride, positions, turns, rot_dims, heads, dk);
  });
  LV_LAUNCH_CHECK();
  p.q = qr; p.k = kr; p.q_stride = p.k_stride = (int64_t)heads * dk;
  const int esize = dtype == LVLLM_F32 ? 4 : 2;
  p.vec_in = ((dv | v_stride | gate_stride) & 3) == 0 && (((uintptr_t)v | (uintptr_t)gate) & (4 * esize - 1)) == 0;
  p.vec_out = ((dv | out_stride) & 3) == 0 && ((uintptr_t)out & (4 * esize - 1)) == 0;
  if (dtype == LVLLM_BF16) launch_mix_sized<BF16, F32, true>(p, s);
  else launch_mix_sized<F32, F32, true>(p, s);
  LV_LAUNCH_CHECK();
  if (p.o == nullptr) return 0;
  return launch_head_norm_gate<true>(out, out_stride, p.o, gate, gate_stride, norm_weight, norm_head_stride, eps, out_scale, rows,
                               heads, dv, dtype, s);
}
