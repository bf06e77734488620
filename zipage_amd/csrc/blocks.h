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

// Sum of squares of each of the block's 16 tokens over the wave's columns; lane l16 == 0 of group g leaves
// tokens 4 g .. 4 g + 3 in `red` (16 floats per wave).
template <int NC> __device__ __forceinline__ void block_squares(const f32x4 (&o)[NC], float* red, int wave) {
  const int l16 = threadIdx.x & 15, g = (threadIdx.x & 63) >> 4;
  f32x4 ss = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int nc = 0; nc < NC; ++nc) ss += o[nc] * o[nc];
#pragma unroll
  for (int r = 0; r < 4; ++r) ss[r] = row16_sum(ss[r]);
  if (l16 == 0) *(f32x4*)(red + wave * kBlock + 4 * g) = ss;
}
template <int NW> __device__ __forceinline__ f32x4 block_squares_total(const float* red) {
  const int g = (threadIdx.x & 63) >> 4;
  f32x4 ss = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int w = 0; w < NW; ++w) ss += *(const f32x4*)(red + w * kBlock + 4 * g);
  return ss;
}

// Forms for 16-bit models on the hardware's exponential, logarithm, reciprocal and reciprocal square root,
// each within a unit or two of the last of 24 bits.
__device__ __forceinline__ float fast_sigmoid(float x) { return __builtin_amdgcn_rcpf(1.f + __expf(-x)); }
__device__ __forceinline__ float fast_softplus(float x) {
  const float y = __expf(-fabsf(x));
  // log(1 + y) as it stands loses a small y's digits
  const float l = y < 0.03125f ? y * (1.f - y * (0.5f - y * (1.f / 3.f - y * 0.25f))) : __logf(1.f + y);
  return fmaxf(x, 0.f) + l;
}

// Element (row 4 g + r, column col) of 16 token rows of bf16, for r = 0 .. 3; rows behind the last read as zero
// and are not written.
struct BlockRows {
  __amdgpu_buffer_rsrc_t rs;
  __device__ __forceinline__ BlockRows(const void* base, int64_t row, int cnt, int64_t stride)
      : rs(__builtin_amdgcn_make_buffer_rsrc((void*)((char*)base + row * stride * 2), 0, (int)(cnt * stride * 2), 0x00020000)) {}
  // as it is in memory: converting it is left to its use, so that nothing waits for the load before
  __device__ __forceinline__ uint16_t ld(int offset, int col) const {
    return __builtin_amdgcn_raw_buffer_load_b16(rs, offset, col * 2, 0);
  }
  __device__ __forceinline__ void st(int offset, int col, float v) const {
    __builtin_amdgcn_raw_buffer_store_b16(float_to_bf16_bits(v), rs, offset, col * 2, 0);
  }
};

// Columns of a 4 x 16 block of 16-bit values in LDS: lane i of a group of sixteen names row i / 4, values 4 (i % 4)
// on, and receives column i.
typedef short s16x4 __attribute__((ext_vector_type(4)));
__device__ __forceinline__ f32x4 read_columns(const char* p) {
  const s16x4 v = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) s16x4*)p);
  return f32x4{bf16_bits_to_float((uint16_t)v[0]), bf16_bits_to_float((uint16_t)v[1]), bf16_bits_to_float((uint16_t)v[2]),
               bf16_bits_to_float((uint16_t)v[3])};
}

// Loads straight into LDS: lane l's 16 bytes from `base` + offset (+ uniform) to `lds` + 16 l.  Written out,
// because the compiler, which cannot tell the stage being filled from the stage being read, would wait for
// them at the next LDS read; wait_and_meet() waits for them.
typedef __attribute__((address_space(3))) void* lds_ptr_t;
struct StageLoads {
  u32x4 rs;
  __device__ __forceinline__ StageLoads(const void* base, int64_t bytes) {
    const uint64_t p = (uint64_t)base;
    rs = u32x4{(uint32_t)__builtin_amdgcn_readfirstlane((int)(uint32_t)p),
               (uint32_t)__builtin_amdgcn_readfirstlane((int)((uint32_t)(p >> 32) & 0xffffu)),
               (uint32_t)__builtin_amdgcn_readfirstlane((int)bytes), 0x00020000u};
  }
  __device__ __forceinline__ void ld(void* lds, int offset, int uniform) const {
    const uint32_t to = (uint32_t)__builtin_amdgcn_readfirstlane((int)(uint32_t)(uintptr_t)(lds_ptr_t)lds);
    const int so = __builtin_amdgcn_readfirstlane(uniform);
    asm volatile("s_mov_b32 m0, %0\n\ts_nop 0\n\tbuffer_load_dwordx4 %1, %2, %3 offen lds"
                 :: "s"(to), "v"(offset), "s"(rs), "s"(so) : "memory", "m0");
  }
};
__device__ __forceinline__ void wait_and_meet() {
  asm volatile("" ::: "memory");
  __builtin_amdgcn_s_waitcnt(0);               // as a builtin: the compiler then knows that nothing is outstanding
  __builtin_amdgcn_s_barrier();
  asm volatile("" ::: "memory");
}

// Blocks of segment i start at slot (row - row0) / 16 + i: enough room, whatever the counts are.
__device__ __forceinline__ int64_t block_slot(int row0, const Segment& sg, int seg, int b) {
  return (sg.row - row0) / kBlock + seg + b;
}

}  // namespace
