// Matrix memory with exponential gates (mLSTM), token by token:
//
//   m' = max(f + m, i);  S' = e^{f + m - m'} S + e^{i - m'} k v^T;  n' likewise with k alone
//   o  = S'^T q / (max(|n' . q|, e^{-m'}) + 1e-6)
//
// with log gates i = cap tanh(./cap), f = logsigmoid(cap tanh(./cap)); then each head's o is divided by
// its root mean square, weighted, and gated by a sigmoid.  One workgroup per (segment, head), state in
// registers, all arithmetic fp32.  Inputs of 16 tokens at a time are staged in LDS; inside a stage
// the waves run without a barrier.
#include "scan.h"

namespace {

template <typename T, int RL, int NW>
__global__ __launch_bounds__(64 * NW) void mlstm_scan_kernel(zp_mlstm a) {
  extern __shared__ __align__(16) float lds[];
  const int dk = a.dk, dv = a.dv;
  float* const qs = lds;                              // [16][dk]
  float* const ks = qs + kScanTokens * dk;            // [16][dk]
  float* const vs = ks + kScanTokens * dk;            // [16][dv]: values, then read-outs
  float* const keep = vs + kScanTokens * dv;          // [16] each
  float* const wr = keep + kScanTokens;
  float* const den = wr + kScanTokens;                // e^{-m}, then the denominator
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, nw = blockDim.x >> 6;
  const int cq = lane_cq(), rg = lane_rg();
  const int h = blockIdx.x % a.heads;
  const Segment sg = segment_of(a.seg, blockIdx.x / a.heads);
  if (sg.count <= 0) {
    if (a.seg.rows == nullptr && sg.row < a.seg.num_rows) clear_rows<T>(a.out, sg.row * a.out_stride + h * dv, a.out_stride, 1, dv);
    return;
  }
  float* const state = a.state + ((int64_t)sg.slot * a.heads + h) * ((int64_t)dk * dv + dk + 4);
  float* const nstate = state + (int64_t)dk * dv;
  const int col = wave * 32 + cq * 4;
  f32x4 S[RL];
#pragma unroll
  for (int r = 0; r < RL; ++r) {
    S[r] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (sg.start > 0) S[r] = *(const f32x4*)(state + (int64_t)(4 * (8 * (r >> 2) + rg) + (r & 3)) * dv + col);
  }
  constexpr int kN = (RL * 8 + 63) / 64;              // normaliser entries per lane of the last wave
  const bool nwave = wave == nw - 1;
  float nv[kN];
#pragma unroll
  for (int j = 0; j < kN; ++j) nv[j] = nwave && sg.start > 0 && lane + 64 * j < dk ? nstate[lane + 64 * j] : 0.f;
  float m = sg.start > 0 ? nstate[dk] : 0.f;
  const float icap = 1.f / a.cap;

  for (int t0 = 0; t0 < sg.count; t0 += kScanTokens) {
    const int cnt = min(kScanTokens, sg.count - t0);
    const int64_t row0 = sg.row + t0;
    const int pk = dk / 8, pv = dv / 8, per = 2 * pk + pv;
    for (int it = tid; it < cnt * per; it += blockDim.x) {
      const int t = it / per, p = it - t * per;
      const int64_t src = (row0 + t) * a.in_stride;
      float x[8];
      if (p < 2 * pk) {
        const bool isq = p < pk;
        const int c = (isq ? p : p - pk) * 8;
        Vec8<T>::ld(a.in, src + (isq ? a.q_at : a.k_at) + h * dk + c, x);
        if (isq) {
#pragma unroll
          for (int i = 0; i < 8; ++i) x[i] *= a.q_scale;
        }
        Vec8<F32>::st((isq ? qs : ks), t * dk + c, x);
      } else {
        const int c = (p - 2 * pk) * 8;
        Vec8<T>::ld(a.in, src + a.v_at + h * dv + c, x);
        Vec8<F32>::st(vs, t * dv + c, x);
      }
    }
    if (wave == 0) {
      float gi = 0.f, gf = 0.f;
      if (lane < cnt) {
        const int64_t src = (row0 + lane) * a.gate_stride + h;
        gi = a.cap * tanhf((a.gates[src] + a.i_bias[h]) * icap);
        const float x = a.cap * tanhf((a.gates[src + a.heads] + a.f_bias[h]) * icap);
        gf = fminf(x, 0.f) - log1pf(expf(-fabsf(x)));
      }
      float before = 0.f, after = 0.f;
      for (int t = 0; t < cnt; ++t) {
        const float ft = __shfl(gf, t), it = __shfl(gi, t);
        const float next = fmaxf(ft + m, it);
        if (lane == t) { before = m; after = next; }
        m = next;
      }
      if (lane < cnt) {
        keep[lane] = expf(gf + before - after);
        wr[lane] = expf(gi - after);
        den[lane] = expf(-after);
      }
    }
    __syncthreads();
    for (int t = 0; t < cnt; ++t) {
      const float kp = keep[t], w = wr[t];
      const f32x4 v = *(const f32x4*)(vs + t * dv + col) * w;
      f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int j = 0; j < RL / 4; ++j) {
        const f32x4 k4 = *(const f32x4*)(ks + t * dk + 4 * (8 * j + rg));
        const f32x4 q4 = *(const f32x4*)(qs + t * dk + 4 * (8 * j + rg));
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          f32x4& s = S[4 * j + i];
#pragma unroll
          for (int c = 0; c < 4; ++c) {
            s[c] = fmaf(k4[i], v[c], s[c] * kp);
            acc[c] = fmaf(s[c], q4[i], acc[c]);
          }
        }
      }
#pragma unroll
      for (int c = 0; c < 4; ++c) acc[c] = rows_sum(acc[c]);
      if (rg == 0) *(f32x4*)(vs + t * dv + col) = acc;
      if (nwave) {
        float d = 0.f;
#pragma unroll
        for (int j = 0; j < kN; ++j) {
          const int r = lane + 64 * j;
          if (r < dk) {
            nv[j] = fmaf(w, ks[t * dk + r], nv[j] * kp);
            d = fmaf(nv[j], qs[t * dk + r], d);
          }
        }
        d = wave_sum(d);
        if (lane == 0) den[t] = fmaxf(fabsf(d), den[t]) + 1e-6f;
      }
    }
    __syncthreads();
    for (int t = wave; t < cnt; t += nw)
      gated_norm_row<T>(vs + t * dv, 1.f / den[t], dv, a.vdim, a.eps, a.norm + h * dv, a.in,
                        (row0 + t) * a.in_stride + a.g_at + h * dv, a.out_scale, a.out,
                        (row0 + t) * a.out_stride + h * dv);
    __syncthreads();
  }
#pragma unroll
  for (int r = 0; r < RL; ++r) *(f32x4*)(state + (int64_t)(4 * (8 * (r >> 2) + rg) + (r & 3)) * dv + col) = S[r];
  if (nwave) {
#pragma unroll
    for (int j = 0; j < kN; ++j)
      if (lane + 64 * j < dk) nstate[lane + 64 * j] = nv[j];
  }
  if (tid == 0) nstate[dk] = m;
}

// One token per segment (decoding): the state passes through once, nothing is staged.
template <typename T, int RL, int NW>
__global__ __launch_bounds__(64 * NW) void mlstm_step_kernel(zp_mlstm a) {
  __shared__ float red[NW];
  const int dk = 8 * RL, dv = a.dv;
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
  const int64_t src = sg.row * a.in_stride + h * dk, vsrc = sg.row * a.in_stride + h * dv + col;
  float* const state = a.state + ((int64_t)sg.slot * a.heads + h) * ((int64_t)dk * dv + dk + 4);
  float* const nstate = state + (int64_t)dk * dv;
  const bool fresh = sg.start == 0;
  constexpr int kN = (RL * 8 + 63) / 64;
  f32x4 S[RL], q[RL / 4], k[RL / 4];
#pragma unroll
  for (int j = 0; j < RL / 4; ++j) {
    q[j] = load4<T>(a.in, src + a.q_at + 4 * (8 * j + rg));
    k[j] = load4<T>(a.in, src + a.k_at + 4 * (8 * j + rg));
  }
  f32x4 v = load4<T>(a.in, vsrc + a.v_at);
  const f32x4 gate = load4<T>(a.in, vsrc + a.g_at);
  float nv[kN], nk[kN], nq[kN];
#pragma unroll
  for (int j = 0; j < kN; ++j) {
    const int c = lane + 64 * j;
    nv[j] = !fresh && c < dk ? nstate[c] : 0.f;
    nk[j] = c < dk ? Elem<T>::ld(a.in, src + a.k_at + c) : 0.f;
    nq[j] = c < dk ? Elem<T>::ld(a.in, src + a.q_at + c) : 0.f;
  }
  const float m0 = fresh ? 0.f : nstate[dk];
  const float zi = a.gates[sg.row * a.gate_stride + h], zf = a.gates[sg.row * a.gate_stride + a.heads + h];
#pragma unroll
  for (int r = 0; r < RL; ++r) {
    S[r] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (!fresh) S[r] = *(const f32x4*)(state + (int64_t)(4 * (8 * (r >> 2) + rg) + (r & 3)) * dv + col);
  }
  const float gi = a.cap * tanhf((zi + a.i_bias[h]) / a.cap), x = a.cap * tanhf((zf + a.f_bias[h]) / a.cap);
  const float gf = fminf(x, 0.f) - log1pf(expf(-fabsf(x)));
  const float m = fmaxf(gf + m0, gi), kp = expf(gf + m0 - m), w = expf(gi - m);
  float d = 0.f;
#pragma unroll
  for (int j = 0; j < kN; ++j) {
    nv[j] = fmaf(w, nk[j], nv[j] * kp);
    d = fmaf(nv[j], nq[j], d);
  }
  d = wave_sum(d) * a.q_scale;
  const float f = a.q_scale / (fmaxf(fabsf(d), expf(-m)) + 1e-6f);
  v *= w;
  f32x4 o = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int r = 0; r < RL; ++r) {
#pragma unroll
    for (int c = 0; c < 4; ++c) {
      S[r][c] = fmaf(k[r >> 2][r & 3], v[c], S[r][c] * kp);
      o[c] = fmaf(S[r][c], q[r >> 2][r & 3], o[c]);
    }
    *(f32x4*)(state + (int64_t)(4 * (8 * (r >> 2) + rg) + (r & 3)) * dv + col) = S[r];
  }
  float ss = 0.f;
#pragma unroll
  for (int c = 0; c < 4; ++c) {
    o[c] = rows_sum(o[c]) * f;
    ss = fmaf(o[c], o[c], ss);
  }
  ss = quads_sum(ss);
  if (lane == 0) red[wave] = ss;
  __syncthreads();                            // also: every wave has read n and m
  ss = 0.f;
  for (int i = 0; i < nw; ++i) ss += red[i];
  const float rs = a.out_scale / sqrtf(ss / (float)a.vdim + a.eps);
  if (rg == 0) {
    const f32x4 wn = *(const f32x4*)(a.norm + h * dv + col);
#pragma unroll
    for (int c = 0; c < 4; ++c) o[c] *= rs * wn[c] * sigmoid_f(gate[c]);
    store4<T>(a.out, out_at, o);
  }
  if (wave == nw - 1) {
#pragma unroll
    for (int j = 0; j < kN; ++j)
      if (lane + 64 * j < dk) nstate[lane + 64 * j] = nv[j];
    if (lane == 0) nstate[dk] = m;
  }
}

template <typename T, int RL> int launch_mlstm(const zp_mlstm& a, hipStream_t st) {
  const size_t smem = sizeof(float) * kScanTokens * (2 * a.dk + a.dv + 3);
  const dim3 grid((unsigned)((int64_t)a.seg.n * a.heads)), block(a.dv * 2);
  if (a.seg.max_count == 1) {
    if (a.dv <= 128) hipLaunchKernelGGL((mlstm_step_kernel<T, RL, 4>), grid, block, 0, st, a);
    else hipLaunchKernelGGL((mlstm_step_kernel<T, RL, 8>), grid, block, 0, st, a);
    ZP_LAUNCH_CHECK();
    return ZP_OK;
  }
  const void* fn = a.dv <= 128 ? (const void*)mlstm_scan_kernel<T, RL, 4> : (const void*)mlstm_scan_kernel<T, RL, 8>;
  if (smem > 64 * 1024 && hipFuncSetAttribute(fn, hipFuncAttributeMaxDynamicSharedMemorySize, (int)smem) != hipSuccess) {
    zp_set_error("mlstm: cannot reserve %zu bytes of LDS", smem);
    return ZP_EHIP;
  }
  if (a.dv <= 128) hipLaunchKernelGGL((mlstm_scan_kernel<T, RL, 4>), grid, block, smem, st, a);
  else hipLaunchKernelGGL((mlstm_scan_kernel<T, RL, 8>), grid, block, smem, st, a);
  ZP_LAUNCH_CHECK();
  return ZP_OK;
}

}  // namespace

extern "C" int zp_mlstm_scan(const zp_mlstm* args, int32_t dtype, void* stream) {
  ZP_REQUIRE(args, "mlstm: null arguments");
  const zp_mlstm& a = *args;
  ZP_REQUIRE(a.seg.n >= 0 && a.heads > 0 && a.vdim > 0 && a.vdim <= a.dv && a.cap > 0.f && a.seg.num_slots > 0 &&
                 a.gate_stride >= 2 * a.heads && a.out_stride >= (int64_t)a.heads * a.dv, "mlstm: bad dims");
  ZP_MODEL_DTYPE("mlstm");
  if ((a.dk != 32 && a.dk != 64 && a.dk != 128 && a.dk != 256) || a.dv % 32 || a.dv > 256 || a.in_stride % 8 ||
      a.q_at % 8 || a.k_at % 8 || a.v_at % 8 || a.g_at % 8 || a.out_stride % 8) {
    zp_set_error("mlstm: head sizes %d (32, 64, 128, 256) and %d (a multiple of 32, <= 256) unsupported", a.dk, a.dv);
    return ZP_EUNSUPPORTED;
  }
  if (a.seg.n == 0) return ZP_OK;
  ZP_REQUIRE(a.in && a.gates && a.i_bias && a.f_bias && a.norm && a.state && a.out && a.seg.counts && a.seg.slots &&
                 a.seg.starts && aligned16(a.in) && aligned16(a.state) && aligned16(a.norm) && aligned16(a.out), "mlstm: null or unaligned pointer");
  hipStream_t st = (hipStream_t)stream;
#define ZP_MLSTM(T)                                    \
  switch (a.dk) {                                      \
    case 32: return launch_mlstm<T, 4>(a, st);         \
    case 64: return launch_mlstm<T, 8>(a, st);         \
    case 128: return launch_mlstm<T, 16>(a, st);       \
    default: return launch_mlstm<T, 32>(a, st);        \
  }
  if (dtype == ZP_BF16) { ZP_MLSTM(BF16); } else { ZP_MLSTM(F32); }
#undef ZP_MLSTM
}
