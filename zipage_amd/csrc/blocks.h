// The recurrent mixers over long runs of tokens: 16 tokens at a time on the fp32 matrix cores, the state
// of a head in registers.
//
// A wave owns 16 * NC columns of the state.  S lies in the result layout of the 16x16 products (lane (g,
// l16) holds rows 16 kt + 4 g + r of column l16 in element r), which is also the layout of a right operand
// if step j of the contraction takes index 4 g + j from lane group g.  So S, and the rows u derived from
// it, enter the next product from the registers they were computed in; left operands give a lane the four
// elements 4 g .. 4 g + 3 of its row.
#pragma once
#include "scan.h"
#include "mfma.h"

namespace {

constexpr int kBlock = 16;

__device__ __forceinline__ f32x4 mfma_f32_step(float a, float b, const f32x4& c) {
  return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0);
}
// c += A B over sixteen of the contraction: a is the left operand's four elements, b a result tile.
__device__ __forceinline__ void mfma_f32_16(const f32x4& a, const f32x4& b, f32x4& c) {
#pragma unroll
  for (int j = 0; j < 4; ++j) c = mfma_f32_step(a[j], b[j], c);
}

template <int KT, int NC> __device__ __forceinline__ void load_state(f32x4 (&S)[KT][NC], const float* state, int dv, int col0, bool fresh) {
  const int l16 = threadIdx.x & 15, g = (threadIdx.x & 63) >> 4;
#pragma unroll
  for (int kt = 0; kt < KT; ++kt)
#pragma unroll
    for (int nc = 0; nc < NC; ++nc)
#pragma unroll
      for (int r = 0; r < 4; ++r)
        S[kt][nc][r] = fresh ? 0.f : state[(int64_t)(16 * kt + 4 * g + r) * dv + col0 + nc * 16 + l16];
}
template <int KT, int NC> __device__ __forceinline__ void store_state(const f32x4 (&S)[KT][NC], float* state, int dv, int col0) {
  const int l16 = threadIdx.x & 15, g = (threadIdx.x & 63) >> 4;
#pragma unroll
  for (int kt = 0; kt < KT; ++kt)
#pragma unroll
    for (int nc = 0; nc < NC; ++nc)
#pragma unroll
      for (int r = 0; r < 4; ++r) state[(int64_t)(16 * kt + 4 * g + r) * dv + col0 + nc * 16 + l16] = S[kt][nc][r];
}

// Sum of squares of each of the block's 16 tokens over the wave's columns; lane l16 == 0 of group g ends
// with tokens 4 g .. 4 g + 3 in `red` (16 floats per wave).
template <int NC> __device__ __forceinline__ void block_squares(const f32x4 (&o)[NC], float* red) {
  const int l16 = threadIdx.x & 15, g = (threadIdx.x & 63) >> 4, wave = threadIdx.x >> 6;
  f32x4 ss = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int nc = 0; nc < NC; ++nc) ss += o[nc] * o[nc];
#pragma unroll
  for (int r = 0; r < 4; ++r) ss[r] = row16_sum(ss[r]);
  if (l16 == 0) *(f32x4*)(red + wave * kBlock + 4 * g) = ss;
}
__device__ __forceinline__ f32x4 block_squares_total(const float* red, int nw) {
  const int g = (threadIdx.x & 63) >> 4;
  f32x4 ss = {0.f, 0.f, 0.f, 0.f};
  for (int w = 0; w < nw; ++w) ss += *(const f32x4*)(red + w * kBlock + 4 * g);
  return ss;
}

}  // namespace
