// Two softmaxes per head over the same values, their difference normed (head_prefill.h, head_decode.h).
#include "head_decode.h"
#include "head_prefill.h"

namespace lvllm {
int launch_head_prefill_maps(const HeadAttnParams& p, hipStream_t s) { return prefill_of_size<2>(p, s); }
int launch_head_decode_maps(const HeadAttnParams& p, hipStream_t s) { return decode_of_size<2>(p, s); }
}  // namespace lvllm
