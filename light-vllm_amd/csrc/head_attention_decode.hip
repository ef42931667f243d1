// Few columns of one softmax per head (head_decode.h).
#include "head_decode.h"

namespace lvllm {
int launch_head_decode(const HeadAttnParams& p, hipStream_t s) { return decode_of_size<1>(p, s); }
}  // namespace lvllm
