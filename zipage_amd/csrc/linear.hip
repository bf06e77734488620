// Linear attention with decay, token by token:
//
//   S <- g * S (rows) + k v^T;  o = S^T q
//
// with a decay per key channel, g = sigmoid(z + bias)^(1/tau), or one fixed decay per head; q and k may turn
// with their position.  Then each head's o is divided by its root mean square, weighted, and gated by a
// silu.  One workgroup per (segment, head), state in registers, all arithmetic fp32: what the products left
// is rotated, decayed and added up without being rounded again.
//
//   linear_scan   portions of any length, 16 tokens staged in LDS at a time
//   linear_step   single tokens (decoding): the state passes through once
#include "linear.h"

namespace {

template <typename T, int RL, int NW>
__global__ __launch_bounds__(64 * NW) void linear_scan_kernel(zp_linear a) {
  extern __shared__ __align__(16) float lds[];
  const int dk = a.dk, dv = a.dv, half = a.rot / 2;
  float* const qs = lds;                              // [16][dk]
  float* const ks = qs + kScanTokens * dk;            // [16][dk]
  float* const gs = ks + kScanTokens * dk;            // [16][dk] decays
  float* const vs = gs + kScanTokens * dk;            // [16][dv]: values, then read-outs
  const int tid = threadIdx.x, wave = tid >> 6, nw = blockDim.x >> 6;
  const int cq = lane_cq(), rg = lane_rg();
  const int h = blockIdx.x % a.heads;
  const Segment sg = segment_of(a.seg, blockIdx.x / a.heads);
  if (sg.count <= 0) {
    if (a.seg.rows == nullptr && sg.row < a.seg.num_rows) clear_rows<T>(a.out, sg.row * a.out_stride + h * dv, a.out_stride, 1, dv);
    return;
  }
  float* const state = a.state + ((int64_t)sg.slot * a.heads + h) * ((int64_t)dk * dv);
  const int col = wave * 32 + cq * 4;
  f32x4 S[RL];
#pragma unroll
  for (int r = 0; r < RL; ++r) {
    S[r] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (sg.start > 0) S[r] = *(const f32x4*)(state + (int64_t)(4 * (8 * (r >> 2) + rg) + (r & 3)) * dv + col);
  }
  for (int t0 = 0; t0 < sg.count; t0 += kScanTokens) {
    const int cnt = min(kScanTokens, sg.count - t0);
    const int64_t row0 = sg.row + t0;
    for (int it = tid; it < cnt * dk; it += blockDim.x) {
      const int t = it / dk, c = it - t * dk;
      const int64_t src = (row0 + t) * a.in_stride + h * dk;
      qs[it] = turned<T>(a, src + a.q_at, c, half, sg.start + t0 + t) * a.q_scale;
      ks[it] = turned<T>(a, src + a.k_at, c, half, sg.start + t0 + t) * a.k_scale;
      gs[it] = a.low ? exact_decay(Elem<T>::ld(a.low, (row0 + t) * a.low_stride + h * dk + c) + a.decay[h * dk + c], a.inv_tau)
                     : a.decay[h];
    }
    for (int it = tid; it < cnt * dv; it += blockDim.x) {
      const int t = it / dv, c = it - t * dv;
      vs[it] = Elem<T>::ld(a.in, (row0 + t) * a.in_stride + a.v_at + h * dv + c);
    }
    __syncthreads();
    for (int t = 0; t < cnt; ++t) {
      const f32x4 v = *(const f32x4*)(vs + t * dv + col);
      f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int j = 0; j < RL / 4; ++j) {
        const int at = t * dk + 4 * (8 * j + rg);
        const f32x4 g4 = *(const f32x4*)(gs + at), k4 = *(const f32x4*)(ks + at), q4 = *(const f32x4*)(qs + at);
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          f32x4& s = S[4 * j + i];
#pragma unroll
          for (int c = 0; c < 4; ++c) {
            s[c] = fmaf(k4[i], v[c], s[c] * g4[i]);
            acc[c] = fmaf(s[c], q4[i], acc[c]);
          }
        }
      }
#pragma unroll
      for (int c = 0; c < 4; ++c) acc[c] = rows_sum(acc[c]);
      if (rg == 0) *(f32x4*)(vs + t * dv + col) = acc;
    }
    __syncthreads();
    for (int t = wave; t < cnt; t += nw)
      gated_norm_row<T, true>(vs + t * dv, 1.f, dv, a.vdim, a.eps, a.norm + h * dv, a.in,
                              (row0 + t) * a.in_stride + a.g_at + h * dv, 1.f, a.out, (row0 + t) * a.out_stride + h * dv);
    __syncthreads();
  }
#pragma unroll
  for (int r = 0; r < RL; ++r) *(f32x4*)(state + (int64_t)(4 * (8 * (r >> 2) + rg) + (r & 3)) * dv + col) = S[r];
}

template <typename T, int RL, int NW>
__global__ __launch_bounds__(64 * NW) void linear_step_kernel(zp_linear a) {
  constexpr int dk = 8 * RL;
  __shared__ __align__(16) float qs[dk], ks[dk], gs[dk];
  __shared__ float red[NW];
  const int dv = a.dv, half = a.rot / 2;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, nw = blockDim.x >> 6;
  const int cq = lane_cq(), rg = lane_rg();
  const int h = blockIdx.x % a.heads;
  const Segment sg = segment_of(a.seg, blockIdx.x / a.heads);
  const int col = wave * 32 + cq * 4;
  const int64_t out_at = sg.row * a.out_stride + h * dv + col;
  if (sg.count <= 0) {
    if (a.seg.rows == nullptr && sg.row < a.seg.num_rows && rg == 0) store4<T>(a.out, out_at, f32x4{0.f, 0.f, 0.f, 0.f});
    return;
  }
  const int64_t src = sg.row * a.in_stride;
  float* const state = a.state + ((int64_t)sg.slot * a.heads + h) * ((int64_t)dk * dv);
  const f32x4 v = load4<T>(a.in, src + a.v_at + h * dv + col), gate = load4<T>(a.in, src + a.g_at + h * dv + col);
  f32x4 S[RL];
#pragma unroll
  for (int r = 0; r < RL; ++r) {
    S[r] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (sg.start > 0) S[r] = *(const f32x4*)(state + (int64_t)(4 * (8 * (r >> 2) + rg) + (r & 3)) * dv + col);
  }
  for (int c = tid; c < dk; c += blockDim.x) {
    qs[c] = turned<T>(a, src + a.q_at + h * dk, c, half, sg.start) * a.q_scale;
    ks[c] = turned<T>(a, src + a.k_at + h * dk, c, half, sg.start) * a.k_scale;
    gs[c] = a.low ? exact_decay(Elem<T>::ld(a.low, sg.row * a.low_stride + h * dk + c) + a.decay[h * dk + c], a.inv_tau) : a.decay[h];
  }
  __syncthreads();
  f32x4 o = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int j = 0; j < RL / 4; ++j) {
    const int at = 4 * (8 * j + rg);
    const f32x4 g4 = *(const f32x4*)(gs + at), k4 = *(const f32x4*)(ks + at), q4 = *(const f32x4*)(qs + at);
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      f32x4& s = S[4 * j + i];
#pragma unroll
      for (int c = 0; c < 4; ++c) {
        s[c] = fmaf(k4[i], v[c], s[c] * g4[i]);
        o[c] = fmaf(s[c], q4[i], o[c]);
      }
      *(f32x4*)(state + (int64_t)(at + i) * dv + col) = s;
    }
  }
  float ss = 0.f;
#pragma unroll
  for (int c = 0; c < 4; ++c) {
    o[c] = rows_sum(o[c]);
    ss = fmaf(o[c], o[c], ss);
  }
  ss = quads_sum(ss);
  if (lane == 0) red[wave] = ss;
  __syncthreads();
  ss = 0.f;
  for (int i = 0; i < nw; ++i) ss += red[i];
  const float rs = 1.f / sqrtf(ss / (float)a.vdim + a.eps);
  if (rg == 0) {
    const f32x4 wn = *(const f32x4*)(a.norm + h * dv + col);
#pragma unroll
    for (int c = 0; c < 4; ++c) o[c] *= rs * wn[c] * gate[c] * sigmoid_f(gate[c]);
    store4<T>(a.out, out_at, o);
  }
}

template <typename T, int RL> int launch_linear(const zp_linear& a, hipStream_t st) {
  const dim3 grid((unsigned)((int64_t)a.seg.n * a.heads)), block(a.dv * 2);
  if (a.seg.max_count == 1) {
    if (a.dv <= 128) hipLaunchKernelGGL((linear_step_kernel<T, RL, 4>), grid, block, 0, st, a);
    else hipLaunchKernelGGL((linear_step_kernel<T, RL, 8>), grid, block, 0, st, a);
    ZP_LAUNCH_CHECK();
    return ZP_OK;
  }
  const size_t smem = sizeof(float) * kScanTokens * (3 * a.dk + a.dv);
  const void* fn = a.dv <= 128 ? (const void*)linear_scan_kernel<T, RL, 4> : (const void*)linear_scan_kernel<T, RL, 8>;
  if (smem > 64 * 1024 && hipFuncSetAttribute(fn, hipFuncAttributeMaxDynamicSharedMemorySize, (int)smem) != hipSuccess) {
    zp_set_error("linear: cannot reserve %zu bytes of LDS", smem);
    return ZP_EHIP;
  }
  if (a.dv <= 128) hipLaunchKernelGGL((linear_scan_kernel<T, RL, 4>), grid, block, smem, st, a);
  else hipLaunchKernelGGL((linear_scan_kernel<T, RL, 8>), grid, block, smem, st, a);
  ZP_LAUNCH_CHECK();
  return ZP_OK;
}

}  // namespace

extern "C" int zp_linear_scan(const zp_linear* args, int32_t dtype, void* stream) {
  ZP_REQUIRE(args, "linear: null arguments");
  const zp_linear& a = *args;
  ZP_REQUIRE(linear_dims_fit(a), "linear: bad dims");
  ZP_MODEL_DTYPE("linear");
  if ((a.dk != 32 && a.dk != 64 && a.dk != 128 && a.dk != 256) || a.dv % 32 || a.dv > 256 || a.in_stride % 8 || a.v_at % 8 ||
      a.g_at % 8 || a.out_stride % 8) {
    zp_set_error("linear: head sizes %d (32, 64, 128, 256) and %d (a multiple of 32, <= 256) unsupported", a.dk, a.dv);
    return ZP_EUNSUPPORTED;
  }
  if (a.seg.n == 0) return ZP_OK;
  ZP_REQUIRE(a.in && a.decay && (a.rot == 0 || a.freqs) && a.norm && a.state && a.out && a.seg.counts && a.seg.slots &&
                 a.seg.starts && aligned16(a.in) && aligned16(a.state) && aligned16(a.norm) && aligned16(a.out),
             "linear: null or unaligned pointer");
  hipStream_t st = (hipStream_t)stream;
#define ZP_LINEAR(T)                                    \
  switch (a.dk) {                                       \
    case 32: return launch_linear<T, 4>(a, st);         \
    case 64: return launch_linear<T, 8>(a, st);         \
    case 128: return launch_linear<T, 16>(a, st);       \
    default: return launch_linear<T, 32>(a, st);        \
  }
  if (dtype == ZP_BF16) { ZP_LINEAR(BF16); } else { ZP_LINEAR(F32); }
#undef ZP_LINEAR
}
