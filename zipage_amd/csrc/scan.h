// What the recurrent mixers share: a step's segments, and how a head's matrix state lies in a workgroup.
#pragma once
#include "models.h"
#include <math.h>

namespace {

typedef zp_f32x4 f32x4;

// A segment is a run of tokens of one sequence in one step: consecutive token rows, a state slot, the
// position of its first token (0: the state starts at zero, whatever the slot holds).
struct Segment {
  int row, count, slot, start;
};
__device__ __forceinline__ Segment segment_of(const zp_segments& s, int i) {
  Segment o;
  o.row = s.rows ? s.rows[i] : i;
  o.count = s.counts[i];
  if (s.max_count > 0) o.count = min(o.count, s.max_count);
  o.slot = s.slots[i];
  o.start = s.starts[i];
  // host-made descriptors: rows and slots outside the buffers are not touched
  if (o.slot < 0 || o.slot >= s.num_slots || o.row < 0 || o.row + o.count > s.num_rows) o.count = 0;
  return o;
}

// The state of a head is a (dk, dv) matrix in fp32.  A wave owns 32 columns: lane (cq, rg) = (lane % 8,
// lane / 8) holds columns 4 cq .. 4 cq + 3 of rows 4 (8 j + rg) .. + 3 for all j < RL / 4, so a load
// instruction covers whole 128-byte lines, and the 16-byte LDS reads of a token's key or query are
// conflict-free broadcasts.
__device__ __forceinline__ int lane_cq() { return threadIdx.x & 7; }
__device__ __forceinline__ int lane_rg() { return (threadIdx.x & 63) >> 3; }

// Sum over the eight row groups, in every lane.
__device__ __forceinline__ float rows_sum(float v) {
  v += dpp_row_ror<8>(v);
  v += lane_xor16(v);
  return v + lane_xor32(v);
}

__device__ __forceinline__ float sigmoid_f(float x) { return 1.f / (1.f + expf(-x)); }
__device__ __forceinline__ float softplus_f(float x) { return fmaxf(x, 0.f) + log1pf(expf(-fabsf(x))); }

// Sum over the eight column quads of a wave (lanes of one row group), in every one of them.
__device__ __forceinline__ float quads_sum(float v) {
  v += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), 0x141, 0xf, 0xf, false));  // half mirror
  v += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), 0xB1, 0xf, 0xf, false));   // [1,0,3,2]
  v += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), 0x4E, 0xf, 0xf, false));   // [2,3,0,1]
  return v;
}

// Four consecutive elements as fp32.
template <typename T> __device__ __forceinline__ f32x4 load4(const void* p, int64_t i);
template <> __device__ __forceinline__ f32x4 load4<BF16>(const void* p, int64_t i) {
  const uint2 v = *(const uint2*)((const uint16_t*)p + i);
  return f32x4{__uint_as_float(v.x << 16), __uint_as_float(v.x & 0xffff0000u), __uint_as_float(v.y << 16),
               __uint_as_float(v.y & 0xffff0000u)};
}
template <> __device__ __forceinline__ f32x4 load4<F32>(const void* p, int64_t i) {
  return *(const f32x4*)((const float*)p + i);
}
template <typename T> __device__ __forceinline__ void store4(void* p, int64_t i, const f32x4& v);
template <> __device__ __forceinline__ void store4<BF16>(void* p, int64_t i, const f32x4& v) {
  const zp_f32x2 a = {v[0], v[1]}, b = {v[2], v[3]};
  uint2 o;
  o.x = __builtin_bit_cast(uint32_t, __builtin_convertvector(a, zp_bf16x2));
  o.y = __builtin_bit_cast(uint32_t, __builtin_convertvector(b, zp_bf16x2));
  *(uint2*)((uint16_t*)p + i) = o;
}
template <> __device__ __forceinline__ void store4<F32>(void* p, int64_t i, const f32x4& v) { *(f32x4*)((float*)p + i) = v; }

constexpr int kScanTokens = 16;   // tokens staged in LDS at a time

// Readout of one token by one wave: o (dv values in LDS, the mean over vdim) normed, weighted, gated by a sigmoid
// or a silu.
template <typename T, bool SILU = false>
__device__ __forceinline__ void gated_norm_row(const float* o, float o_scale, int dv, int vdim, float eps,
                                               const float* w, const void* gate, int64_t gate_at, float scale,
                                               void* out, int64_t out_at) {
  const int lane = threadIdx.x & 63;
  float ss = 0.f;
  for (int c = lane; c < dv; c += 64) {
    const float x = o[c] * o_scale;
    ss += x * x;
  }
  ss = wave_sum(ss);
  const float rs = scale / sqrtf(ss / (float)vdim + eps) * o_scale;
  for (int c = lane; c < dv; c += 64) {
    const float z = Elem<T>::ld(gate, gate_at + c);
    Elem<T>::st(out, out_at + c, o[c] * rs * w[c] * (SILU ? z * sigmoid_f(z) : sigmoid_f(z)));
  }
}

template <typename T>
__device__ __forceinline__ void clear_rows(void* out, int64_t at, int64_t stride, int count, int dv) {
  for (int t = 0; t < count; ++t)
    for (int c = threadIdx.x; c < dv; c += blockDim.x) Elem<T>::st(out, at + t * stride + c, 0.f);
}

}  // namespace
