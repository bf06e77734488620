// Linear attention with decay: what its token-by-token and its blocked form share.
#pragma once
#include "scan.h"

namespace {

// sigmoid(z)^(1/tau)
__device__ __forceinline__ float exact_decay(float z, float inv_tau) { return expf(-softplus_f(-z) * inv_tau); }

// Channel c of a head's query or key at element `at`, turned by its position: c < half with c + half.
template <typename T> __device__ __forceinline__ float turned(const zp_linear& a, int64_t at, int c, int half, int position) {
  const float x = Elem<T>::ld(a.in, at + c);
  if (c >= 2 * half) return x;
  const int i = c < half ? c : c - half;
  const float2 r = rotary_turn(position, a.freqs[i]);
  const float y = Elem<T>::ld(a.in, at + (c < half ? c + half : i));
  return c < half ? x * r.x - y * r.y : x * r.x + y * r.y;
}

inline bool linear_dims_fit(const zp_linear& a) {
  return a.seg.n >= 0 && a.heads > 0 && a.vdim > 0 && a.vdim <= a.dv && a.rot >= 0 && a.rot % 2 == 0 && a.rot <= a.dk &&
         a.seg.num_slots > 0 && a.out_stride >= (int64_t)a.heads * a.dv && (!a.low || a.low_stride >= (int64_t)a.heads * a.dk) &&
         a.q_at >= 0 && a.k_at >= 0 && a.v_at >= 0 && a.g_at >= 0 &&
         a.in_stride >= (int64_t)a.heads * a.dk + (a.q_at > a.k_at ? a.q_at : a.k_at) &&
         a.in_stride >= (int64_t)a.heads * a.dv + (a.v_at > a.g_at ? a.v_at : a.g_at);
}

}  // namespace
