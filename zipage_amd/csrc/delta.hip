// Gated delta rule with one decay per key channel, token by token:
//
//   S <- g * S (rows);  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q
//
// q, k, v are short causal convolutions of their projections (one filter per channel, silu), q and k
// unit vectors per head, g = exp(-e^{A} softplus(a + bias)), beta a sigmoid; then each head's o is
// divided by its root mean square, weighted, and gated by a sigmoid.  One workgroup per (segment,
// head), state in registers, all arithmetic fp32.  Everything between the projections and the output
// projection is this one launch: the convolutions of 16 tokens at a time are staged in LDS.  Each value
// head keeps the last inputs of its own convolutions, also of the query / key channels it shares, so
// no workgroup writes what another one reads.
#include "scan.h"

namespace {

constexpr int kMaxTaps = 8;

template <typename T, int RL, int NW>
__global__ __launch_bounds__(64 * NW) void delta_scan_kernel(zp_delta a) {
  extern __shared__ __align__(16) float lds[];
  const int dk = a.dk, dv = a.dv, taps = a.taps;
  float* const qs = lds;                              // [16][dk]
  float* const ks = qs + kScanTokens * dk;            // [16][dk]
  float* const gs = ks + kScanTokens * dk;            // [16][dk] decays
  float* const vs = gs + kScanTokens * dk;            // [16][dv]: values, then read-outs
  float* const beta = vs + kScanTokens * dv;          // [16] each
  float* const kq = beta + kScanTokens;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, nw = blockDim.x >> 6;
  const int cq = lane_cq(), rg = lane_rg();
  const int h = blockIdx.x % a.heads, hk = h / (a.heads / a.kv_heads);
  const Segment sg = segment_of(a.seg, blockIdx.x / a.heads);
  if (sg.count <= 0) {
    if (a.seg.rows == nullptr && sg.row < a.seg.num_rows) clear_rows<T>(a.out, sg.row * a.out_stride + h * dv, a.out_stride, 1, dv);
    return;
  }
  const int64_t item = (int64_t)sg.slot * a.heads + h;
  float* const state = a.state + item * ((int64_t)dk * dv);
  const int cw = 2 * dk + dv;                         // channels of the head: q, k, v
  char* const tail = (char*)a.conv_state + item * (taps - 1) * cw * T::bytes;
  const int col = wave * 32 + cq * 4;
  f32x4 S[RL];
#pragma unroll
  for (int r = 0; r < RL; ++r) {
    S[r] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (sg.start > 0) S[r] = *(const f32x4*)(state + (int64_t)(4 * (8 * (r >> 2) + rg) + (r & 3)) * dv + col);
  }
  const float rate = expf(a.a_log[h]);
  const int channels = 2 * a.kv_heads * dk + a.heads * dv;
  // channel c of the head: where it is in a projected row, and among the filters
  auto place = [&](int c) -> int {
    return c < dk ? hk * dk + c : (c < 2 * dk ? a.kv_heads * dk + hk * dk + c - dk : 2 * a.kv_heads * dk + h * dv + c - 2 * dk);
  };
  // input u of channel c, u counted from the segment's first token
  auto input = [&](int u, int c, int at) -> float {
    if (u >= 0) return Elem<T>::ld(a.in, (int64_t)(sg.row + u) * a.in_stride + at);
    return sg.start > 0 ? Elem<T>::ld(tail, (int64_t)(taps - 1 + u) * cw + c) : 0.f;
  };
  auto conv = [&](int u, int c) -> float {
    const int at = place(c);
    float y = 0.f;
    for (int j = 0; j < taps; ++j) y = fmaf(a.filters[(int64_t)j * channels + at], input(u - taps + 1 + j, c, at), y);
    return y * sigmoid_f(y);
  };

  for (int t0 = 0; t0 < sg.count; t0 += kScanTokens) {
    const int cnt = min(kScanTokens, sg.count - t0);
    const int64_t row0 = sg.row + t0;
    for (int t = wave; t < cnt; t += nw) {
      float qv[(RL * 8 + 63) / 64], kv[(RL * 8 + 63) / 64], q2 = 0.f, k2 = 0.f, qk = 0.f;
#pragma unroll
      for (int j = 0; j < (RL * 8 + 63) / 64; ++j) {
        const int c = lane + 64 * j;
        qv[j] = kv[j] = 0.f;
        if (c < dk) {
          qv[j] = conv(t0 + t, c);
          kv[j] = conv(t0 + t, dk + c);
          const float z = Elem<T>::ld(a.low, (row0 + t) * a.low_stride + h * dk + c) + a.dt_bias[h * dk + c];
          gs[t * dk + c] = expf(-rate * softplus_f(z));
        }
        q2 = fmaf(qv[j], qv[j], q2);
        k2 = fmaf(kv[j], kv[j], k2);
        qk = fmaf(qv[j], kv[j], qk);
      }
      const float rq = a.q_scale / sqrtf(wave_sum(q2) + 1e-6f), rk = 1.f / sqrtf(wave_sum(k2) + 1e-6f);
      qk = wave_sum(qk);
#pragma unroll
      for (int j = 0; j < (RL * 8 + 63) / 64; ++j) {
        const int c = lane + 64 * j;
        if (c < dk) {
          qs[t * dk + c] = qv[j] * rq;
          ks[t * dk + c] = kv[j] * rk;
        }
      }
      for (int c = lane; c < dv; c += 64) vs[t * dv + c] = conv(t0 + t, 2 * dk + c);
      if (lane == 0) {
        kq[t] = qk * rq * rk;
        beta[t] = sigmoid_f(Elem<T>::ld(a.in, (row0 + t) * a.in_stride + a.b_at + h));
      }
    }
    __syncthreads();
    for (int t = 0; t < cnt; ++t) {
      const f32x4 v = *(const f32x4*)(vs + t * dv + col);
      f32x4 ak = {0.f, 0.f, 0.f, 0.f}, aq = ak;
#pragma unroll
      for (int j = 0; j < RL / 4; ++j) {
        const int at = t * dk + 4 * (8 * j + rg);
        const f32x4 g4 = *(const f32x4*)(gs + at), k4 = *(const f32x4*)(ks + at), q4 = *(const f32x4*)(qs + at);
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          f32x4& s = S[4 * j + i];
#pragma unroll
          for (int c = 0; c < 4; ++c) {
            s[c] *= g4[i];
            ak[c] = fmaf(s[c], k4[i], ak[c]);
            aq[c] = fmaf(s[c], q4[i], aq[c]);
          }
        }
      }
      const float b = beta[t], x = kq[t];
      f32x4 u;
#pragma unroll
      for (int c = 0; c < 4; ++c) {
        u[c] = b * (v[c] - rows_sum(ak[c]));
        aq[c] = fmaf(u[c], x, rows_sum(aq[c]));         // the read-out sees this token's write
      }
#pragma unroll
      for (int j = 0; j < RL / 4; ++j) {
        const f32x4 k4 = *(const f32x4*)(ks + t * dk + 4 * (8 * j + rg));
#pragma unroll
        for (int i = 0; i < 4; ++i)
#pragma unroll
          for (int c = 0; c < 4; ++c) S[4 * j + i][c] = fmaf(k4[i], u[c], S[4 * j + i][c]);
      }
      if (rg == 0) *(f32x4*)(vs + t * dv + col) = aq;
    }
    __syncthreads();
    for (int t = wave; t < cnt; t += nw)
      gated_norm_row<T>(vs + t * dv, 1.f, dv, a.vdim, a.eps, a.norm + h * dv, a.low,
                        (row0 + t) * a.low_stride + a.g_at + h * dv, a.out_scale, a.out,
                        (row0 + t) * a.out_stride + h * dv);
    __syncthreads();
  }
#pragma unroll
  for (int r = 0; r < RL; ++r) *(f32x4*)(state + (int64_t)(4 * (8 * (r >> 2) + rg) + (r & 3)) * dv + col) = S[r];
  for (int c = tid; c < cw; c += blockDim.x) {
    const int at = place(c);
    float last[kMaxTaps];
#pragma unroll
    for (int e = 0; e < kMaxTaps; ++e)
      if (e < taps - 1) last[e] = input(sg.count - (taps - 1) + e, c, at);
#pragma unroll
    for (int e = 0; e < kMaxTaps; ++e)
      if (e < taps - 1) Elem<T>::st(tail, (int64_t)e * cw + c, last[e]);
  }
}

// One token per segment (decoding): the state passes through once.
template <typename T, int RL, int NW>
__global__ __launch_bounds__(64 * NW) void delta_step_kernel(zp_delta a) {
  extern __shared__ __align__(16) float lds[];
  __shared__ float red[NW];
  const int dk = 8 * RL, dv = a.dv, taps = a.taps, cw = 2 * dk + dv;
  float* const qs = lds;                              // convolved q, k, v, then decays
  float* const ks = qs + dk;
  float* const vs = ks + dk;
  float* const gs = vs + dv;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, nw = blockDim.x >> 6;
  const int cq = lane_cq(), rg = lane_rg();
  const int h = blockIdx.x % a.heads, hk = h / (a.heads / a.kv_heads);
  const Segment sg = segment_of(a.seg, blockIdx.x / a.heads);
  const int col = wave * 32 + cq * 4;
  const int64_t out_at = sg.row * a.out_stride + h * dv + col;
  if (sg.count <= 0) {
    if (a.seg.rows == nullptr && sg.row < a.seg.num_rows && rg == 0) store4<T>(a.out, out_at, f32x4{0.f, 0.f, 0.f, 0.f});
    return;
  }
  const int64_t item = (int64_t)sg.slot * a.heads + h;
  float* const state = a.state + item * ((int64_t)dk * dv);
  char* const tail = (char*)a.conv_state + item * (taps - 1) * cw * T::bytes;
  const int channels = 2 * a.kv_heads * dk + a.heads * dv;
  const bool fresh = sg.start == 0;
  const int64_t src = sg.row * a.in_stride;
  auto place = [&](int c) -> int {
    return c < dk ? hk * dk + c : (c < 2 * dk ? a.kv_heads * dk + hk * dk + c - dk : 2 * a.kv_heads * dk + h * dv + c - 2 * dk);
  };
  // a channel's last inputs, its filter and its place in the history, which moves on by one
  struct Taps { float x[kMaxTaps], f[kMaxTaps]; };
  auto fetch = [&](int c, Taps& o) {
    const int at = place(c);
#pragma unroll
    for (int e = 0; e < kMaxTaps; ++e) {
      o.x[e] = o.f[e] = 0.f;
      if (e < taps) {
        o.f[e] = a.filters[(int64_t)e * channels + at];
        o.x[e] = e == taps - 1 ? Elem<T>::ld(a.in, src + at) : (fresh ? 0.f : Elem<T>::ld(tail, (int64_t)e * cw + c));
      }
    }
  };
  auto finish = [&](int c, const Taps& o) {
    float y = 0.f;
#pragma unroll
    for (int e = 0; e < kMaxTaps; ++e) y = fmaf(o.f[e], o.x[e], y);
    lds[c] = y * sigmoid_f(y);
#pragma unroll
    for (int e = 1; e < kMaxTaps; ++e)
      if (e < taps) Elem<T>::st(tail, (int64_t)(e - 1) * cw + c, o.x[e]);
  };
  Taps first, second;
  if (tid < cw) fetch(tid, first);
  const int c2 = tid + blockDim.x;
  if (c2 < cw) fetch(c2, second);
  float z = 0.f;
  if (tid < dk) z = Elem<T>::ld(a.low, sg.row * a.low_stride + h * dk + tid) + a.dt_bias[h * dk + tid];
  const float zb = Elem<T>::ld(a.in, src + a.b_at + h), rate = expf(a.a_log[h]);
  const f32x4 gate = load4<T>(a.low, sg.row * a.low_stride + a.g_at + h * dv + col);
  f32x4 S[RL];
#pragma unroll
  for (int r = 0; r < RL; ++r) {
    S[r] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (!fresh) S[r] = *(const f32x4*)(state + (int64_t)(4 * (8 * (r >> 2) + rg) + (r & 3)) * dv + col);
  }
  if (tid < cw) finish(tid, first);
  if (c2 < cw) finish(c2, second);
  for (int c = c2 + blockDim.x; c < cw; c += blockDim.x) {
    fetch(c, first);
    finish(c, first);
  }
  if (tid < dk) gs[tid] = expf(-rate * softplus_f(z));
  for (int c = tid + blockDim.x; c < dk; c += blockDim.x)
    gs[c] = expf(-rate * softplus_f(Elem<T>::ld(a.low, sg.row * a.low_stride + h * dk + c) + a.dt_bias[h * dk + c]));
  __syncthreads();
  float q2 = 0.f, k2 = 0.f, qk = 0.f;
  for (int c = lane; c < dk; c += 64) {
    const float q = qs[c], k = ks[c];
    q2 = fmaf(q, q, q2);
    k2 = fmaf(k, k, k2);
    qk = fmaf(q, k, qk);
  }
  const float rq = a.q_scale / sqrtf(wave_sum(q2) + 1e-6f), rk = 1.f / sqrtf(wave_sum(k2) + 1e-6f);
  qk = wave_sum(qk) * rq * rk;
  f32x4 ak = {0.f, 0.f, 0.f, 0.f}, aq = ak, k4[RL / 4];
#pragma unroll
  for (int j = 0; j < RL / 4; ++j) {
    const int at = 4 * (8 * j + rg);
    const f32x4 g4 = *(const f32x4*)(gs + at), q4 = *(const f32x4*)(qs + at) * rq;
    k4[j] = *(const f32x4*)(ks + at) * rk;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      f32x4& s = S[4 * j + i];
#pragma unroll
      for (int c = 0; c < 4; ++c) {
        s[c] *= g4[i];
        ak[c] = fmaf(s[c], k4[j][i], ak[c]);
        aq[c] = fmaf(s[c], q4[i], aq[c]);
      }
    }
  }
  const f32x4 v = *(const f32x4*)(vs + col);
  const float b = sigmoid_f(zb);
  f32x4 u;
  float ss = 0.f;
#pragma unroll
  for (int c = 0; c < 4; ++c) {
    u[c] = b * (v[c] - rows_sum(ak[c]));
    aq[c] = fmaf(u[c], qk, rows_sum(aq[c]));            // the read-out sees this token's write
    ss = fmaf(aq[c], aq[c], ss);
  }
#pragma unroll
  for (int r = 0; r < RL; ++r) {
#pragma unroll
    for (int c = 0; c < 4; ++c) S[r][c] = fmaf(k4[r >> 2][r & 3], u[c], S[r][c]);
    *(f32x4*)(state + (int64_t)(4 * (8 * (r >> 2) + rg) + (r & 3)) * dv + col) = S[r];
  }
  ss = quads_sum(ss);
  if (lane == 0) red[wave] = ss;
  __syncthreads();
  ss = 0.f;
  for (int i = 0; i < nw; ++i) ss += red[i];
  const float rs = a.out_scale / sqrtf(ss / (float)a.vdim + a.eps);
  if (rg == 0) {
    const f32x4 wn = *(const f32x4*)(a.norm + h * dv + col);
#pragma unroll
    for (int c = 0; c < 4; ++c) aq[c] *= rs * wn[c] * sigmoid_f(gate[c]);
    store4<T>(a.out, out_at, aq);
  }
}

template <typename T, int RL> int launch_delta(const zp_delta& a, hipStream_t st) {
  const size_t smem = sizeof(float) * kScanTokens * (3 * a.dk + a.dv + 2);
  const dim3 grid((unsigned)((int64_t)a.seg.n * a.heads)), block(a.dv * 2);
  if (a.seg.max_count == 1) {
    const size_t step = sizeof(float) * (3 * a.dk + a.dv);
    if (a.dv <= 128) hipLaunchKernelGGL((delta_step_kernel<T, RL, 4>), grid, block, step, st, a);
    else hipLaunchKernelGGL((delta_step_kernel<T, RL, 8>), grid, block, step, st, a);
    ZP_LAUNCH_CHECK();
    return ZP_OK;
  }
  const void* fn = a.dv <= 128 ? (const void*)delta_scan_kernel<T, RL, 4> : (const void*)delta_scan_kernel<T, RL, 8>;
  if (smem > 64 * 1024 && hipFuncSetAttribute(fn, hipFuncAttributeMaxDynamicSharedMemorySize, (int)smem) != hipSuccess) {
    zp_set_error("delta: cannot reserve %zu bytes of LDS", smem);
    return ZP_EHIP;
  }
  if (a.dv <= 128) hipLaunchKernelGGL((delta_scan_kernel<T, RL, 4>), grid, block, smem, st, a);
  else hipLaunchKernelGGL((delta_scan_kernel<T, RL, 8>), grid, block, smem, st, a);
  ZP_LAUNCH_CHECK();
  return ZP_OK;
}

}  // namespace

extern "C" int zp_delta_scan(const zp_delta* args, int32_t dtype, void* stream) {
  ZP_REQUIRE(args, "delta: null arguments");
  const zp_delta& a = *args;
  ZP_REQUIRE(a.seg.n >= 0 && a.heads > 0 && a.kv_heads > 0 && a.heads % a.kv_heads == 0 && a.vdim > 0 && a.vdim <= a.dv &&
                 a.seg.num_slots > 0 && a.out_stride >= (int64_t)a.heads * a.dv, "delta: bad dims");
  ZP_MODEL_DTYPE("delta");
  if ((a.dk != 32 && a.dk != 64 && a.dk != 128 && a.dk != 256) || a.dv % 32 || a.dv > 256 || a.taps < 1 || a.taps > kMaxTaps ||
      a.low_stride % 8 || a.g_at % 8 || a.out_stride % 8) {
    zp_set_error("delta: head sizes %d (32, 64, 128, 256) and %d (a multiple of 32, <= 256), %d taps (1 .. %d) unsupported",
                 a.dk, a.dv, a.taps, kMaxTaps);
    return ZP_EUNSUPPORTED;
  }
  if (a.seg.n == 0) return ZP_OK;
  ZP_REQUIRE(a.in && a.low && a.filters && a.a_log && a.dt_bias && a.norm && a.state && (a.conv_state || a.taps == 1) && a.out &&
                 a.seg.counts && a.seg.slots && a.seg.starts && aligned16(a.state) && aligned16(a.norm) && aligned16(a.low) &&
                 aligned16(a.out), "delta: null or unaligned pointer");
  hipStream_t st = (hipStream_t)stream;
#define ZP_DELTA(T)                                    \
  switch (a.dk) {                                      \
    case 32: return launch_delta<T, 4>(a, st);         \
    case 64: return launch_delta<T, 8>(a, st);         \
    case 128: return launch_delta<T, 16>(a, st);       \
    default: return launch_delta<T, 32>(a, st);        \
  }
  if (dtype == ZP_BF16) { ZP_DELTA(BF16); } else { ZP_DELTA(F32); }
#undef ZP_DELTA
}
