// Device helpers shared by the model-side kernels that exist in bfloat16 and in float32.
#pragma once
#include "common.h"
#include "../../include/zipage_models.h"
#include <math.h>

#define ZP_MODEL_DTYPE(name)                                       \
  if (dtype != ZP_BF16 && dtype != ZP_F32) {                       \
    zp_set_error(name ": bfloat16 and float32 only");              \
    return ZP_EUNSUPPORTED;                                        \
  }

static inline bool aligned16(const void* p) { return (uintptr_t)p % 16 == 0; }

typedef uint32_t zp_u32x4 __attribute__((ext_vector_type(4)));
typedef float zp_f32x4 __attribute__((ext_vector_type(4)));

// Eight consecutive elements as fp32, 16-byte accesses; `i` is a multiple of 8.
// Or in two steps, so that nothing waits for the load before its use: raw() and unpack().
template <typename T> struct Vec8;
template <> struct Vec8<BF16> {
  typedef zp_u32x4 Raw;
  __device__ static __forceinline__ Raw raw(const void* p, int64_t i) { return *(const zp_u32x4*)((const uint16_t*)p + i); }
  __device__ static __forceinline__ void ld(const void* p, int64_t i, float* o) { unpack(raw(p, i), o); }
  __device__ static __forceinline__ void unpack(const Raw& v, float* o) {
#pragma unroll
    for (int k = 0; k < 4; ++k) {
      o[2 * k] = __uint_as_float(v[k] << 16);
      o[2 * k + 1] = __uint_as_float(v[k] & 0xffff0000u);
    }
  }
  __device__ static __forceinline__ void st(void* p, int64_t i, const float* o) {
    zp_u32x4 v;
#pragma unroll
    for (int k = 0; k < 4; ++k) {
      const zp_f32x2 f = {o[2 * k], o[2 * k + 1]};
      v[k] = __builtin_bit_cast(uint32_t, __builtin_convertvector(f, zp_bf16x2));
    }
    *(zp_u32x4*)((uint16_t*)p + i) = v;
  }
};
template <> struct Vec8<F32> {
  struct Raw { zp_f32x4 a, b; };
  __device__ static __forceinline__ Raw raw(const void* p, int64_t i) {
    return Raw{*(const zp_f32x4*)((const float*)p + i), *(const zp_f32x4*)((const float*)p + i + 4)};
  }
  __device__ static __forceinline__ void ld(const void* p, int64_t i, float* o) { unpack(raw(p, i), o); }
  __device__ static __forceinline__ void unpack(const Raw& v, float* o) {
#pragma unroll
    for (int k = 0; k < 4; ++k) { o[k] = v.a[k]; o[k + 4] = v.b[k]; }
  }
  __device__ static __forceinline__ void st(void* p, int64_t i, const float* o) {
    *(zp_f32x4*)((float*)p + i) = zp_f32x4{o[0], o[1], o[2], o[3]};
    *(zp_f32x4*)((float*)p + i + 4) = zp_f32x4{o[4], o[5], o[6], o[7]};
  }
};

// tanh; in 16-bit models on the hardware's exponential and reciprocal (absolute error below 2e-7, relative
// below 2e-5).
__device__ __forceinline__ float fast_tanh(float x) {
  const float t = __builtin_amdgcn_exp2f(-2.88539008177793f * fabsf(x));      // exp(-2 |x|)
  const float big = copysignf((1.f - t) * __builtin_amdgcn_rcpf(1.f + t), x);
  const float q = x * x;                          // near zero the difference above loses digits
  return fabsf(x) < 0.0625f ? x * (1.f - q * (1.f / 3.f - q * (2.f / 15.f))) : big;
}
// Scores of 16-bit attention in powers of two: log2(e) scale x, under a soft cap log2(e) cap tanh(scale x / cap).
// The cap's tanh is 1 - 2 / (1 + exp(2 z)), whose error is a rounding of the cap, not of the score.  A cap that
// keeps the powers far inside fp32's range makes a running maximum unnecessary (`bounded`).
__host__ __device__ inline bool soft_cap_bounded(float cap) { return cap > 0.f && cap * 1.44269504088896f <= 80.f; }
struct SoftCap {
  float factor, top;
  bool on, bounded;
  __device__ __forceinline__ SoftCap(float scale, float cap)
      : factor(cap > 0.f ? scale / cap * 2.88539008177793f : scale * 1.44269504088896f), top(cap * 1.44269504088896f),
        on(cap > 0.f), bounded(soft_cap_bounded(cap)) {}
  __device__ __forceinline__ float capped(float x) const {
    return fmaf(-2.f * top, __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(x * factor)), top);
  }
  __device__ __forceinline__ float log2_score(float x) const { return on ? capped(x) : x * factor; }
};

template <typename T> __device__ __forceinline__ float tanh_of(float x);
template <> __device__ __forceinline__ float tanh_of<F32>(float x) { return tanhf(x); }
template <> __device__ __forceinline__ float tanh_of<BF16>(float x) { return fast_tanh(x); }
template <typename T> __device__ __forceinline__ float sigmoid_of(float x);
template <> __device__ __forceinline__ float sigmoid_of<F32>(float x) { return 1.f / (1.f + expf(-x)); }
template <> __device__ __forceinline__ float sigmoid_of<BF16>(float x) { return __builtin_amdgcn_rcpf(1.f + __expf(-x)); }

// Angles of rotary positions are fp32: position times frequency.
__device__ __forceinline__ float2 rotary_turn(int position, float freq) {
  float s, c;
  sincosf((float)position * freq, &s, &c);
  return make_float2(c, s);
}
// A pair turns by an angle.
__device__ __forceinline__ void turn_pair(float& u, float& v, float c, float s) {
  const float x = u, y = v;
  u = x * c - y * s;
  v = y * c + x * s;
}
// Eight elements, adjacent ones a pair, turn back by the angles of four (cos, sin).
__device__ __forceinline__ void turn_back8(float* r, const float2* t) {
  const zp_f32x4 a = ((const zp_f32x4*)t)[0], b = ((const zp_f32x4*)t)[1];
  turn_pair(r[0], r[1], a[0], -a[1]);
  turn_pair(r[2], r[3], a[2], -a[3]);
  turn_pair(r[4], r[5], b[0], -b[1]);
  turn_pair(r[6], r[7], b[2], -b[3]);
}
