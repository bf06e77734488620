// Gated delta rule (delta.hip) over long runs, 16 tokens at a time.  With G_t the product of the block's
// decays up to token t, per key channel, a block is
//
//   A[t, s] = beta_t sum_c k_t k_s G_t / G_s (s < t),   P[t, s] = sum_c q_t k_s G_t / G_s (s <= t)
//   (1 + A) [U0 | W] = beta [V | G k],   U = U0 - W S,   O = (G q) S + P U
//   S <- G_15 S + sum_s (G_15 / G_s) k_s u_s^T
//
// delta_prepare computes everything without S for all blocks at once and leaves it in the order of the
// matrix operands; ratios of decays are running products of the decays themselves, so nothing is divided
// and nothing overflows.  delta_blocks walks a head's blocks with S in registers.  All fp32.
#include "blocks.h"

namespace {

constexpr int kMaxTaps = 8;

struct RunArgs {
  zp_delta d;
  float* ws;
  int row0;      // first token row of the first segment
};

__host__ __device__ inline int block_floats(int dk, int dv) { return kBlock * (3 * dk + dv) + kBlock * kBlock + dk; }
// Blocks of segment i start at slot (row - row0) / 16 + i: enough room, whatever the counts are.
__device__ __forceinline__ int64_t block_slot(const RunArgs& a, const Segment& sg, int seg, int b) {
  return (sg.row - a.row0) / kBlock + seg + b;
}

template <typename T>
__global__ __launch_bounds__(256) void delta_prepare_kernel(RunArgs ra) {
  extern __shared__ __align__(16) float lds[];
  const zp_delta& a = ra.d;
  const int dk = a.dk, dv = a.dv, taps = a.taps;
  const Segment sg = segment_of(a.seg, blockIdx.z);
  const int t0 = blockIdx.x * kBlock;
  if (t0 >= sg.count || sg.row < ra.row0) return;
  const int cnt = min(kBlock, sg.count - t0);
  const int h = blockIdx.y, hk = h / (a.heads / a.kv_heads);
  float* const qs = lds;                       // [16][dk]
  float* const ks = qs + kBlock * dk;
  float* const gs = ks + kBlock * dk;
  float* const vs = gs + kBlock * dk;          // [16][dv]
  float* const As = vs + kBlock * dv;          // [16][16]
  float* const Ps = As + kBlock * kBlock;      // [16][16]
  float* const beta = Ps + kBlock * kBlock;
  float* const outs = beta + kBlock;           // W and G q in operand order, 4 floats of padding per 64
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int cw = 2 * dk + dv;
  const char* const tail = (const char*)a.conv_state + ((int64_t)sg.slot * a.heads + h) * (taps - 1) * cw * T::bytes;
  const float rate = expf(a.a_log[h]);
  const int channels = 2 * a.kv_heads * dk + a.heads * dv;
  auto place = [&](int c) -> int {
    return c < dk ? hk * dk + c : (c < 2 * dk ? a.kv_heads * dk + hk * dk + c - dk : 2 * a.kv_heads * dk + h * dv + c - 2 * dk);
  };
  // ---- convolutions: a thread's channel, the block's 16 tokens from a sliding window
  for (int c = tid; c < cw; c += 256) {
    const int at = place(c);
    float x[kBlock + kMaxTaps - 1], f[kMaxTaps];
#pragma unroll
    for (int j = 0; j < kMaxTaps; ++j) f[j] = j < taps ? a.filters[(int64_t)(taps - 1 - j) * channels + at] : 0.f;   // f[j]: j tokens back
#pragma unroll
    for (int i = 0; i < kBlock + kMaxTaps - 1; ++i) {
      const int u = t0 + i - (kMaxTaps - 1);
      x[i] = 0.f;
      if (i >= kMaxTaps - taps && u < t0 + cnt) {
        if (u >= 0) x[i] = Elem<T>::ld(a.in, (int64_t)(sg.row + u) * a.in_stride + at);
        else if (sg.start > 0) x[i] = Elem<T>::ld(tail, (int64_t)(taps - 1 + u) * cw + c);
      }
    }
    float* const dst = c < dk ? qs + c : (c < 2 * dk ? ks + c - dk : vs + c - 2 * dk);
    const int st = c < 2 * dk ? dk : dv;
#pragma unroll
    for (int t = 0; t < kBlock; ++t) {
      float y = 0.f;
#pragma unroll
      for (int j = 0; j < kMaxTaps; ++j) y = fmaf(f[j], x[t + kMaxTaps - 1 - j], y);
      dst[t * st] = t < cnt ? y * sigmoid_f(y) : 0.f;
    }
  }
  for (int i = tid; i < kBlock * dk; i += 256) {
    const int t = i / dk, c = i - t * dk;
    float g = 1.f;
    if (t < cnt) {
      const float z = Elem<T>::ld(a.low, (int64_t)(sg.row + t0 + t) * a.low_stride + h * dk + c) + a.dt_bias[h * dk + c];
      g = expf(-rate * softplus_f(z));
    }
    gs[i] = g;
  }
  if (tid < kBlock)
    beta[tid] = tid < cnt ? sigmoid_f(Elem<T>::ld(a.in, (int64_t)(sg.row + t0 + tid) * a.in_stride + a.b_at + h)) : 0.f;
  __syncthreads();
  // ---- unit vectors: a wave its four tokens
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int t = wave * 4 + i;
    float q2 = 0.f, k2 = 0.f;
    for (int c = lane; c < dk; c += 64) {
      const float q = qs[t * dk + c], k = ks[t * dk + c];
      q2 = fmaf(q, q, q2);
      k2 = fmaf(k, k, k2);
    }
    const float rq = a.q_scale / sqrtf(wave_sum(q2) + 1e-6f), rk = 1.f / sqrtf(wave_sum(k2) + 1e-6f);
    for (int c = lane; c < dk; c += 64) {
      qs[t * dk + c] *= rq;
      ks[t * dk + c] *= rk;
    }
  }
  __syncthreads();
  // ---- A and P: lane group (lane / 16) of wave w walks k_s, s = 4 w + group, down the tokens; 16 lanes share
  // its channels in pieces of four
  {
    const int l16 = lane & 15, s = wave * 4 + (lane >> 4), pieces = dk / 4;
    f32x4 kk[2];
#pragma unroll
    for (int p = 0; p < 2; ++p) {
      const int pc = l16 + 16 * p;
      kk[p] = f32x4{0.f, 0.f, 0.f, 0.f};
      if (pc < pieces) kk[p] = *(const f32x4*)(ks + s * dk + pc * 4);
    }
#pragma unroll
    for (int t = 0; t < kBlock; ++t) {
      float sa = 0.f, sp = 0.f;
      if (t >= wave * 4) {                    // uniform in the wave
#pragma unroll
        for (int p = 0; p < 2; ++p) {
          const int pc = l16 + 16 * p;
          if (pc < pieces) {
            if (t > s) kk[p] *= *(const f32x4*)(gs + t * dk + pc * 4);
            const f32x4 kt = *(const f32x4*)(ks + t * dk + pc * 4), qt = *(const f32x4*)(qs + t * dk + pc * 4);
#pragma unroll
            for (int i = 0; i < 4; ++i) {
              sa = fmaf(kk[p][i], kt[i], sa);
              sp = fmaf(kk[p][i], qt[i], sp);
            }
          }
        }
        sa = row16_sum(sa);
        sp = row16_sum(sp);
      }
      if (l16 == 0) {
        As[t * kBlock + s] = t > s ? sa * beta[t] : 0.f;
        Ps[t * kBlock + s] = t >= s ? sp : 0.f;
      }
    }
  }
  __syncthreads();
  // ---- columns: forward substitution, and the block's decays
  const int64_t base = (block_slot(ra, sg, blockIdx.z, blockIdx.x) * a.heads + h) * block_floats(dk, dv);
  float* const oWQ = ra.ws + base;             // [2][dk / 16][64 lanes][4]
  float* const oK = oWQ + 2 * kBlock * dk;     // [dk / 16][64][4]
  float* const oU = oK + kBlock * dk;          // [dv / 16][64][4]
  float* const oP = oU + kBlock * dv;          // [64][4]
  float* const oG = oP + kBlock * kBlock;      // [dk]
  for (int c = tid; c < dk + dv; c += 256) {
    float w[kBlock];
    if (c < dk) {
      float G = 1.f;
      const int at = (c >> 4) * 272 + ((c & 15) >> 2) * 68 + (c & 3);      // 256 and 64 floats, padded
#pragma unroll
      for (int t = 0; t < kBlock; ++t) {
        G *= gs[t * dk + c];
        w[t] = beta[t] * ks[t * dk + c] * G;
        outs[(dk / 16) * 272 + at + t * 4] = qs[t * dk + c] * G;
      }
      oG[c] = G;
    } else {
#pragma unroll
      for (int t = 0; t < kBlock; ++t) w[t] = beta[t] * vs[t * dv + c - dk];
    }
#pragma unroll
    for (int t = 1; t < kBlock; ++t) {
#pragma unroll
      for (int s = 0; s < t; ++s) w[t] = fmaf(-As[t * kBlock + s], w[s], w[t]);
    }
    if (c < dk) {
      const int at = (c >> 4) * 272 + ((c & 15) >> 2) * 68 + (c & 3);
#pragma unroll
      for (int t = 0; t < kBlock; ++t) outs[at + t * 4] = -w[t];
      float R = 1.f;
#pragma unroll
      for (int t = kBlock - 1; t >= 0; --t) {
        w[t] = ks[t * dk + c] * R;
        R *= gs[t * dk + c];
      }
#pragma unroll
      for (int g = 0; g < 4; ++g)
        *(f32x4*)(oK + ((c >> 4) * 64 + g * 16 + (c & 15)) * 4) = f32x4{w[4 * g], w[4 * g + 1], w[4 * g + 2], w[4 * g + 3]};
    } else {
      const int v = c - dk;
#pragma unroll
      for (int g = 0; g < 4; ++g)
        *(f32x4*)(oU + ((v >> 4) * 64 + g * 16 + (v & 15)) * 4) = f32x4{w[4 * g], w[4 * g + 1], w[4 * g + 2], w[4 * g + 3]};
    }
  }
  if (tid < 64) *(f32x4*)(oP + tid * 4) = *(const f32x4*)(Ps + (tid & 15) * kBlock + (tid >> 4) * 4);
  __syncthreads();
  for (int i = tid; i < 2 * kBlock * dk / 4; i += 256) {
    const int x = i * 4, tile = x >> 8, in = x & 255;
    *(f32x4*)(oWQ + x) = *(const f32x4*)(outs + tile * 272 + (in >> 6) * 68 + (in & 63));
  }
}

template <typename T, int KT, int NC>
__global__ __launch_bounds__(NC == 2 ? 256 : 512) void delta_blocks_kernel(RunArgs ra) {
  const zp_delta& a = ra.d;
  __shared__ float red[2][16 * kBlock];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, nw = blockDim.x >> 6, l16 = lane & 15, g = lane >> 4;
  const int dk = 16 * KT, dv = a.dv;
  const int h = blockIdx.x % a.heads, seg = blockIdx.x / a.heads;
  const Segment sg = segment_of(a.seg, seg);
  if (sg.count <= 0 || sg.row < ra.row0) return;
  const int64_t item = (int64_t)sg.slot * a.heads + h;
  float* const state = a.state + item * ((int64_t)dk * dv);
  const int col0 = wave * 16 * NC;
  f32x4 S[KT][NC];
  load_state<KT, NC>(S, state, dv, col0, sg.start == 0);
  float nrm[NC];
#pragma unroll
  for (int nc = 0; nc < NC; ++nc) nrm[nc] = a.norm[h * dv + col0 + nc * 16 + l16] * a.out_scale;
  const int64_t stride = (int64_t)a.heads * block_floats(dk, dv);
  const float* blk = ra.ws + (block_slot(ra, sg, seg, 0) * a.heads + h) * block_floats(dk, dv) + lane * 4;
  const int blocks = (sg.count + kBlock - 1) / kBlock;
  f32x4 W[KT], Q[KT], U[NC];
  auto fetch = [&](const float* p) {
#pragma unroll
    for (int kt = 0; kt < KT; ++kt) {
      W[kt] = *(const f32x4*)(p + kt * 256);
      Q[kt] = *(const f32x4*)(p + (KT + kt) * 256);
    }
#pragma unroll
    for (int nc = 0; nc < NC; ++nc) U[nc] = *(const f32x4*)(p + 3 * kBlock * dk + (wave * NC + nc) * 256);
  };
  fetch(blk);
  for (int b = 0; b < blocks; ++b, blk += stride) {
    f32x4 K[KT];
#pragma unroll
    for (int kt = 0; kt < KT; ++kt) K[kt] = *(const f32x4*)(blk + (2 * KT + kt) * 256);
    const f32x4 P = *(const f32x4*)(blk + kBlock * (3 * dk + dv));
    const float* const dec = blk - lane * 4 + kBlock * (3 * dk + dv) + kBlock * kBlock + 4 * g;
    const int cnt = min(kBlock, sg.count - b * kBlock);
    const int64_t row = sg.row + b * kBlock;
    float gate[NC][4];
#pragma unroll
    for (int nc = 0; nc < NC; ++nc)
#pragma unroll
      for (int r = 0; r < 4; ++r)
        gate[nc][r] = Elem<T>::ld(a.low, (row + min(4 * g + r, cnt - 1)) * a.low_stride + a.g_at + h * dv + col0 + nc * 16 + l16);
    f32x4 O[NC];
#pragma unroll
    for (int nc = 0; nc < NC; ++nc) O[nc] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int kt = 0; kt < KT; ++kt)
#pragma unroll
      for (int j = 0; j < 4; ++j)
#pragma unroll
        for (int nc = 0; nc < NC; ++nc) {
          U[nc] = mfma_f32_step(W[kt][j], S[kt][nc][j], U[nc]);
          O[nc] = mfma_f32_step(Q[kt][j], S[kt][nc][j], O[nc]);
        }
#pragma unroll
    for (int nc = 0; nc < NC; ++nc) mfma_f32_16(P, U[nc], O[nc]);
    f32x4 u[NC];
#pragma unroll
    for (int nc = 0; nc < NC; ++nc) u[nc] = U[nc];
    fetch(b + 1 < blocks ? blk + stride : blk);
#pragma unroll
    for (int kt = 0; kt < KT; ++kt) {
      const f32x4 d = *(const f32x4*)(dec + 16 * kt);
#pragma unroll
      for (int nc = 0; nc < NC; ++nc) {
        S[kt][nc] *= d;
        mfma_f32_16(K[kt], u[nc], S[kt][nc]);
      }
    }
    block_squares<NC>(O, red[b & 1]);
    __syncthreads();
    const f32x4 ss = block_squares_total(red[b & 1], nw);
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const float rs = 1.f / sqrtf(ss[r] / (float)a.vdim + a.eps);
      if (4 * g + r < cnt) {
#pragma unroll
        for (int nc = 0; nc < NC; ++nc)
          Elem<T>::st(a.out, (row + 4 * g + r) * a.out_stride + h * dv + col0 + nc * 16 + l16,
                      O[nc][r] * rs * nrm[nc] * sigmoid_f(gate[nc][r]));
      }
    }
  }
  store_state<KT, NC>(S, state, dv, col0);
  // the last inputs of the head's convolutions (runs are longer than a filter)
  const int taps = a.taps, cw = 2 * dk + dv, hk = h / (a.heads / a.kv_heads);
  char* const tail = (char*)a.conv_state + item * (taps - 1) * cw * T::bytes;
  for (int i = tid; i < (taps - 1) * cw; i += blockDim.x) {
    const int e = i / cw, c = i - e * cw;
    const int at = c < dk ? hk * dk + c : (c < 2 * dk ? a.kv_heads * dk + hk * dk + c - dk : 2 * a.kv_heads * dk + h * dv + c - 2 * dk);
    Elem<T>::st(tail, i, Elem<T>::ld(a.in, (int64_t)(sg.row + max(sg.count - (taps - 1) + e, 0)) * a.in_stride + at));
  }
}

template <typename T, int KT> int launch_blocks(const RunArgs& ra, hipStream_t st) {
  const zp_delta& a = ra.d;
  const unsigned grid = (unsigned)((int64_t)a.seg.n * a.heads);
  // few heads: half the columns per wave, twice the waves
  const bool narrow = (int64_t)grid * (a.dv / 32) < 1024;
  if (narrow) hipLaunchKernelGGL((delta_blocks_kernel<T, KT, 1>), dim3(grid), dim3(a.dv * 4), 0, st, ra);
  else hipLaunchKernelGGL((delta_blocks_kernel<T, KT, 2>), dim3(grid), dim3(a.dv * 2), 0, st, ra);
  ZP_LAUNCH_CHECK();
  return ZP_OK;
}

template <typename T> int launch_runs(const RunArgs& ra, int longest, hipStream_t st) {
  const zp_delta& a = ra.d;
  const size_t smem = sizeof(float) * (kBlock * (3 * a.dk + a.dv) + 2 * kBlock * kBlock + kBlock + 2 * (a.dk / 16) * 272);
  if (smem > 64 * 1024 && hipFuncSetAttribute((const void*)delta_prepare_kernel<T>, hipFuncAttributeMaxDynamicSharedMemorySize,
                                              (int)smem) != hipSuccess) {
    zp_set_error("delta_runs: cannot reserve %zu bytes of LDS", smem);
    return ZP_EHIP;
  }
  hipLaunchKernelGGL((delta_prepare_kernel<T>), dim3((unsigned)((longest + kBlock - 1) / kBlock), (unsigned)a.heads, (unsigned)a.seg.n),
                     dim3(256), smem, st, ra);
  ZP_LAUNCH_CHECK();
  switch (a.dk) {
    case 32: return launch_blocks<T, 2>(ra, st);
    case 64: return launch_blocks<T, 4>(ra, st);
    default: return launch_blocks<T, 8>(ra, st);
  }
}

}  // namespace

extern "C" int64_t zp_delta_runs_workspace(int32_t rows, int32_t segments, int32_t heads, int32_t dk, int32_t dv) {
  if (rows < 0 || segments < 0 || heads <= 0 || dk <= 0 || dv <= 0) return -1;
  return ((int64_t)rows / kBlock + segments) * heads * block_floats(dk, dv) * 4;
}

extern "C" int zp_delta_runs(const zp_delta* args, int32_t first_row, int32_t longest, void* workspace,
                             int64_t workspace_bytes, int32_t dtype, void* stream) {
  ZP_REQUIRE(args, "delta_runs: null arguments");
  const zp_delta& a = *args;
  ZP_REQUIRE(a.seg.n >= 0 && a.heads > 0 && a.kv_heads > 0 && a.heads % a.kv_heads == 0 && a.vdim > 0 && a.vdim <= a.dv &&
                 a.seg.num_slots > 0 && a.out_stride >= (int64_t)a.heads * a.dv && first_row >= 0 && longest >= 0 &&
                 first_row <= a.seg.num_rows, "delta_runs: bad dims");
  ZP_MODEL_DTYPE("delta_runs");
  if ((a.dk != 32 && a.dk != 64 && a.dk != 128) || a.dv % 32 || a.dv > 128 || a.taps < 1 || a.taps > kMaxTaps || a.heads > 65535 ||
      a.seg.n > 65535) {
    zp_set_error("delta_runs: head sizes %d (32, 64, 128) and %d (a multiple of 32, <= 128), %d taps (1 .. %d) unsupported",
                 a.dk, a.dv, a.taps, kMaxTaps);
    return ZP_EUNSUPPORTED;
  }
  if (a.seg.n == 0 || longest == 0) return ZP_OK;
  ZP_REQUIRE(a.in && a.low && a.filters && a.a_log && a.dt_bias && a.norm && a.state && (a.conv_state || a.taps == 1) && a.out &&
                 a.seg.rows && a.seg.counts && a.seg.slots && a.seg.starts && aligned16(a.state) && aligned16(workspace),
             "delta_runs: null or unaligned pointer");
  ZP_REQUIRE(workspace && workspace_bytes >= zp_delta_runs_workspace(a.seg.num_rows - first_row, a.seg.n, a.heads, a.dk, a.dv),
             "delta_runs: workspace too small");
  RunArgs ra = {a, (float*)workspace, first_row};
  ra.d.seg.max_count = longest;               // no segment has more blocks than were prepared
  return dtype == ZP_BF16 ? launch_runs<BF16>(ra, longest, (hipStream_t)stream) : launch_runs<F32>(ra, longest, (hipStream_t)stream);
}
