// Shared by the general-head-size attention kernels (attn_gd_prefill.hip, attn_gd_decode.hip).
#pragma once
#include "common.h"
#include "kernels.h"

namespace oamd {
namespace gd {

typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef __bf16 bf16x4 __attribute__((ext_vector_type(4)));
typedef short s16x4 __attribute__((ext_vector_type(4)));
typedef float f32x8 __attribute__((ext_vector_type(8)));

__device__ __forceinline__ bf16x8 bf8(u16x8 v) { return __builtin_bit_cast(bf16x8, v); }

// smallest instantiated head size >= d (multiples of 32 up to 256), or -1
inline int dim_bin(int d) {
  if (d <= 32) return 32;
  if (d <= 64) return 64;
  if (d <= 96) return 96;
  if (d <= 128) return 128;
  if (d <= 192) return 192;
  return d <= 256 ? 256 : -1;
}

}  // namespace gd
}  // namespace oamd
