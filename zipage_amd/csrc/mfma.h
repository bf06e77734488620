// bf16 matrix-core helpers of the attention kernels.
#pragma once
#include "models.h"
#include <math.h>

namespace {

typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef zp_u32x4 u32x4;
typedef zp_f32x4 f32x4;

__device__ __forceinline__ f32x4 mfma_bf16(const u32x4& a, const u32x4& b, const f32x4& c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, a),
                                                 __builtin_bit_cast(bf16x8, b), c, 0, 0, 0);
}
__device__ __forceinline__ uint32_t pack_bf16(float lo, float hi) {
  const zp_f32x2 f = {lo, hi};
  return __builtin_bit_cast(uint32_t, __builtin_convertvector(f, zp_bf16x2));
}
// key of operand element i (0..7) held by lane group g, within a step of 32 keys
__device__ __forceinline__ int step_key(int g, int i) { return i < 4 ? 4 * g + i : 12 + 4 * g + i; }

// Eight rows (keys) of eight bf16 columns -> for column t the four dwords of its eight keys.
__device__ __forceinline__ u32x4 column_of(const u32x4* rows, int t) {
  const uint32_t sel = (t & 1) ? 0x07060302u : 0x05040100u;
  u32x4 o;
#pragma unroll
  for (int d = 0; d < 4; ++d)
    o[d] = __builtin_amdgcn_perm(rows[2 * d + 1][t >> 1], rows[2 * d][t >> 1], sel);
  return o;
}

}  // namespace
