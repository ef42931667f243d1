// Chunks of one softmax per head (head_prefill.h).
#include "head_prefill.h"

namespace lvllm {
int launch_head_prefill(const HeadAttnParams& p, hipStream_t s) { return prefill_of_size<1>(p, s); }
}  // namespace lvllm
