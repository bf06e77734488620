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

constexpr int kScanTokens = 16;   // tokens staged in LDS at a time

// Readout of one token by one wave: o (dv values in LDS, the mean over vdim) normed, weighted, gated.
template <typename T>
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
  for (int c = lane; c < dv; c += 64)
    Elem<T>::st(out, out_at + c, o[c] * rs * w[c] * sigmoid_f(Elem<T>::ld(gate, gate_at + c)));
}

template <typename T>
__device__ __forceinline__ void clear_rows(void* out, int64_t at, int64_t stride, int count, int dv) {
  for (int t = 0; t < count; ++t)
    for (int c = threadIdx.x; c < dv; c += blockDim.x) Elem<T>::st(out, at + t * stride + c, 0.f);
}

}  // namespace
