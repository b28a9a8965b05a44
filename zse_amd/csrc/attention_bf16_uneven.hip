// The matrix-core attention for heads whose values are half or twice as wide as their keys (see
// attention_bf16.hip, which chooses the kernels and has the entry points).
#include "attention_bf16_kernels.h"

#if ZSE_ACT_BF16

int attn_launch_uneven(int what, const AttnParams& p, dim3 grid, hipStream_t s) {
#define PAIR_OF_SIZES(H, V) \
  if (p.hd == 16 * H && p.vd == 16 * V) return launch_sizes<H, V>(what, p, grid, s);
  PAIR_OF_SIZES(1, 2)
  PAIR_OF_SIZES(2, 4)
  PAIR_OF_SIZES(4, 8)
  PAIR_OF_SIZES(8, 16)
  PAIR_OF_SIZES(2, 1)
  PAIR_OF_SIZES(4, 2)
  PAIR_OF_SIZES(8, 4)
  PAIR_OF_SIZES(16, 8)
#undef PAIR_OF_SIZES
  return zk_fail("zk_attention_bf16: values as wide as keys, half or twice as wide");
}

#endif  // ZSE_ACT_BF16
