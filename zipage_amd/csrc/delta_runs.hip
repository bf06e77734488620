// Gated delta rule (delta.hip) over long runs, 16 tokens at a time.  With G_t the product of the block's
// decays up to token t, per key channel, a block is
//
//   A[t, s] = beta_t sum_c k_t k_s G_t / G_s (s < t),   P[t, s] = sum_c q_t k_s G_t / G_s (s <= t)
//   (1 + A) [U0 | W] = beta [V | G k],   U = U0 - W S,   O = (G q) S + P U
//   S <- G_15 S + sum_s (G_15 / G_s) k_s u_s^T
//
// delta_prepare computes everything without S for all blocks at once and leaves it in the order of the
// matrix operands; ratios of decays are running products of the decays themselves, so nothing is divided
// and nothing overflows.  delta_blocks walks a head's blocks with S in registers.  All fp32; projections in
// bfloat16.
#include "blocks.h"

namespace {

constexpr int kMaxTaps = 8;

struct RunArgs {
  zp_delta d;
  float* ws;
  int row0;      // first token row of the first segment
};

// [-W | G q] and the keys as left operands, U0 as a result tile, P, the block's decays; whole KBs
__host__ __device__ inline constexpr int block_floats(int dk, int dv) {
  return (kBlock * (3 * dk + dv) + kBlock * kBlock + dk + 255) / 256 * 256;
}

template <int TAPS>
__global__ __launch_bounds__(256, 4) void delta_prepare_kernel(RunArgs ra) {
  extern __shared__ __align__(16) float lds[];
  const zp_delta& a = ra.d;
  constexpr int ld = 132;                      // every row: reads across tokens meet no conflicts, offsets are constants
  const int dk = a.dk, dv = a.dv, taps = a.taps;
  const Segment sg = segment_of(a.seg, blockIdx.z);
  const int t0 = blockIdx.x * kBlock;
  if (t0 >= sg.count || sg.row < ra.row0) return;
  const int cnt = min(kBlock, sg.count - t0);
  const int h = blockIdx.y, hk = h / (a.heads / a.kv_heads);
  float* const qs = lds;                       // [16][ld], later G q
  float* const ks = qs + kBlock * ld;
  float* const gs = ks + kBlock * ld;          // decays, later -W
  float* const vs = gs + kBlock * ld;
  float* const As = vs + kBlock * ld;          // [16][16]
  float* const Ps = As + kBlock * kBlock;      // [16][16]
  float* const beta = Ps + kBlock * kBlock;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int cw = 2 * dk + dv;
  const char* const tail = (const char*)a.conv_state + ((int64_t)sg.slot * a.heads + h) * (taps - 1) * cw * 2;
  const int channels = 2 * a.kv_heads * dk + a.heads * dv;
  auto place = [&](int c) -> int {
    return c < dk ? hk * dk + c : (c < 2 * dk ? a.kv_heads * dk + hk * dk + c - dk : 2 * a.kv_heads * dk + h * dv + c - 2 * dk);
  };
  // ---- requests first: the decays' pre-activations (two pieces a thread at most), the step sizes'
  f32x4 z[2], zb[2];
#pragma unroll
  for (int u = 0; u < 2; ++u) {
    const int i = tid + u * 256, t = i / (dk / 4), c = (i - t * (dk / 4)) * 4;
    z[u] = zb[u] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (t < cnt) {
      z[u] = load4<BF16>(a.low, (int64_t)(sg.row + t0 + t) * a.low_stride + h * dk + c);
      zb[u] = *(const f32x4*)(a.dt_bias + h * dk + c);
    }
  }
  const float b_in = tid < cnt ? Elem<BF16>::ld(a.in, (int64_t)(sg.row + t0 + tid) * a.in_stride + a.b_at + h) : 0.f;
  const float rate = __expf(a.a_log[h]);
  // ---- convolutions: a thread's two channels, the block's 16 tokens from a sliding window
  // rows from t0 - (TAPS - 1) on; those outside the run read as zero, those before it come from the history
  const int back = min(TAPS - 1, t0);
  const __amdgpu_buffer_rsrc_t rows = __builtin_amdgcn_make_buffer_rsrc(
      (void*)((const char*)a.in + (int64_t)(sg.row + t0 - back) * a.in_stride * 2), 0, (int)((cnt + back) * a.in_stride * 2), 0x00020000);
  for (int c = 2 * tid; c < cw; c += 512) {
    const int at = place(c);
    uint32_t x[kBlock + TAPS - 1];             // two channels' bf16
#pragma unroll
    for (int i = 0; i < kBlock + TAPS - 1; ++i) {
      const int u = i - (TAPS - 1) + back;     // row of the buffer
      x[i] = u >= 0 ? (uint32_t)__builtin_amdgcn_raw_buffer_load_b32(rows, at * 2, u * (int)a.in_stride * 2, 0) : 0u;
    }
    if (t0 == 0 && sg.start > 0) {
#pragma unroll
      for (int i = 0; i < TAPS - 1; ++i)
        if (i >= TAPS - taps) x[i] = *(const uint32_t*)(tail + ((int64_t)(taps - TAPS + i) * cw + c) * 2);
    }
    float f[2][TAPS];
#pragma unroll
    for (int j = 0; j < TAPS; ++j)                            // f[.][j]: j tokens back
#pragma unroll
      for (int e = 0; e < 2; ++e) f[e][j] = j < taps ? a.filters[(int64_t)(taps - 1 - j) * channels + at + e] : 0.f;
    float* const dst = c < dk ? qs + c : (c < 2 * dk ? ks + c - dk : vs + c - 2 * dk);
#pragma unroll
    for (int t = 0; t < kBlock; ++t) {
      float2 y = {0.f, 0.f};
#pragma unroll
      for (int j = 0; j < TAPS; ++j) {
        const uint32_t v = x[t + TAPS - 1 - j];
        y.x = fmaf(f[0][j], __uint_as_float(v << 16), y.x);
        y.y = fmaf(f[1][j], __uint_as_float(v & 0xffff0000u), y.y);
      }
      y.x = t < cnt ? y.x * fast_sigmoid(y.x) : 0.f;
      y.y = t < cnt ? y.y * fast_sigmoid(y.y) : 0.f;
      *(float2*)(dst + t * ld) = y;
      if (t % 4 == 3) __builtin_amdgcn_sched_barrier(0);
    }
  }
#pragma unroll
  for (int u = 0; u < 2; ++u) {
    const int i = tid + u * 256, t = i / (dk / 4), c = (i - t * (dk / 4)) * 4;
    if (t < kBlock) {
      f32x4 g = {1.f, 1.f, 1.f, 1.f};
      if (t < cnt) {
#pragma unroll
        for (int e = 0; e < 4; ++e) g[e] = __expf(-rate * fast_softplus(z[u][e] + zb[u][e]));
      }
      *(f32x4*)(gs + t * ld + c) = g;
    }
  }
  if (tid < kBlock) beta[tid] = tid < cnt ? fast_sigmoid(b_in) : 0.f;
  __syncthreads();
  // ---- unit vectors: a wave its four tokens, 16 lanes each
  {
    const int t = wave * 4 + (lane >> 4), l16 = lane & 15, pieces = dk / 4;
    f32x4 q[2], k[2], q2 = {0.f, 0.f, 0.f, 0.f}, k2 = q2;
#pragma unroll
    for (int p = 0; p < 2; ++p) {
      const int pc = min(l16 + 16 * p, pieces - 1);
      q[p] = *(const f32x4*)(qs + t * ld + pc * 4);
      k[p] = *(const f32x4*)(ks + t * ld + pc * 4);
      if (l16 + 16 * p < pieces) {
        q2 += q[p] * q[p];
        k2 += k[p] * k[p];
      }
    }
    const float rq = a.q_scale / sqrtf(row16_sum(q2[0] + q2[1] + q2[2] + q2[3]) + 1e-6f);
    const float rk = 1.f / sqrtf(row16_sum(k2[0] + k2[1] + k2[2] + k2[3]) + 1e-6f);
#pragma unroll
    for (int p = 0; p < 2; ++p) {
      const int pc = l16 + 16 * p;
      if (pc < pieces) {
        *(f32x4*)(qs + t * ld + pc * 4) = q[p] * rq;
        *(f32x4*)(ks + t * ld + pc * 4) = k[p] * rk;
      }
    }
  }
  __syncthreads();
  // ---- A and P: 16 lanes walk k_s down the tokens, in pieces of four channels; group i of wave w takes s = w + 4 i
  {
    const int l16 = lane & 15, s = wave + 4 * (lane >> 4), pieces = dk / 4;
    int at[2];
    f32x4 kk[2];
#pragma unroll
    for (int p = 0; p < 2; ++p) {
      const int pc = l16 + 16 * p;
      at[p] = min(pc, pieces - 1) * 4;
      kk[p] = *(const f32x4*)(ks + s * ld + at[p]);
      if (pc >= pieces) kk[p] = f32x4{0.f, 0.f, 0.f, 0.f};
    }
#pragma unroll
    for (int t = 0; t < kBlock; ++t) {
      f32x4 pa = {0.f, 0.f, 0.f, 0.f}, pp = pa;
#pragma unroll
      for (int p = 0; p < 2; ++p) {
        const f32x4 gt = *(const f32x4*)(gs + t * ld + at[p]);
#pragma unroll
        for (int e = 0; e < 4; ++e) kk[p][e] *= t > s ? gt[e] : 1.f;
        pa += kk[p] * *(const f32x4*)(ks + t * ld + at[p]);
        pp += kk[p] * *(const f32x4*)(qs + t * ld + at[p]);
      }
      const float sa = row16_sum((pa[0] + pa[1]) + (pa[2] + pa[3])), sp = row16_sum((pp[0] + pp[1]) + (pp[2] + pp[3]));
      As[t * kBlock + s] = t > s ? sa * beta[t] : 0.f;         // all 16 lanes, the same value
      Ps[t * kBlock + s] = t >= s ? sp : 0.f;
      if (t % 2 == 1) __builtin_amdgcn_sched_barrier(0);       // not all tokens' rows in registers at once
    }
  }
  __syncthreads();
  // ---- columns: forward substitution, and the block's decays.  A thread reads and writes its own column only.
  const int64_t base = (block_slot(ra.row0, sg, blockIdx.z, blockIdx.x) * a.heads + h) * block_floats(dk, dv);
  float* const oWQ = ra.ws + base;             // [2][dk / 16][64 lanes][4]
  float* const oK = oWQ + 2 * kBlock * dk;     // [dk / 16][64][4]
  float* const oU = oK + kBlock * dk;          // [dv / 16][64][4]
  float* const oP = oU + kBlock * dv;          // [64][4]
  float* const oG = oP + kBlock * kBlock;      // [dk]
  float w[kBlock];
  auto substitute = [&](int t, float b) {      // w_t = b - sum_{s < t} A[t, s] w_s
    float x[4] = {b, 0.f, 0.f, 0.f};
#pragma unroll
    for (int s = 0; s < t; s += 4) {
      const f32x4 A = *(const f32x4*)(As + t * kBlock + s);
#pragma unroll
      for (int i = 0; i < 4; ++i)
        if (s + i < t) x[i] = fmaf(-A[i], w[s + i], x[i]);
    }
    w[t] = (x[0] + x[1]) + (x[2] + x[3]);
    if (t % 2 == 1) __builtin_amdgcn_sched_barrier(0);
  };
  for (int c = tid; c < dk; c += 256) {
    float G = 1.f;
#pragma unroll
    for (int t = 0; t < kBlock; ++t) {
      G *= gs[t * ld + c];
      qs[t * ld + c] *= G;
      substitute(t, beta[t] * ks[t * ld + c] * G);
    }
    oG[c] = G;
    asm volatile("" ::: "memory");            // keys and decays are read again rather than kept
    float R = 1.f;
#pragma unroll
    for (int g = 3; g >= 0; --g) {
      f32x4 x;
#pragma unroll
      for (int r = 3; r >= 0; --r) {
        const int t = 4 * g + r;
        x[r] = ks[t * ld + c] * R;
        R *= gs[t * ld + c];
        gs[t * ld + c] = -w[t];
      }
      *(f32x4*)(oK + ((c >> 4) * 64 + g * 16 + (c & 15)) * 4) = x;
      __builtin_amdgcn_sched_barrier(0);
    }
  }
  for (int v = (tid + 256 - dk) % 256; v < dv; v += 256) {      // on the threads the keys leave free, as far as they go
#pragma unroll
    for (int t = 0; t < kBlock; ++t) substitute(t, beta[t] * vs[t * ld + v]);
#pragma unroll
    for (int g = 0; g < 4; ++g)
      *(f32x4*)(oU + ((v >> 4) * 64 + g * 16 + (v & 15)) * 4) = f32x4{w[4 * g], w[4 * g + 1], w[4 * g + 2], w[4 * g + 3]};
  }
  if (tid < 64) *(f32x4*)(oP + tid * 4) = *(const f32x4*)(Ps + (tid & 15) * kBlock + (tid >> 4) * 4);
  __syncthreads();
  for (int i = tid; i < 2 * kBlock * dk / 4; i += 256) {       // lane (g, row) of tile kt: columns 16 kt + 4 g ..
    const int tile = i >> 6, l = i & 63, kt = tile & (dk / 16 - 1);
    *(f32x4*)(oWQ + i * 4) = *(const f32x4*)((tile < dk / 16 ? gs : qs) + (l & 15) * ld + kt * 16 + (l >> 4) * 4);
  }
}

// A head's blocks, one after the other: a block's operands come straight into LDS while the block before it is
// worked on; its rows are normed and stored behind the next meeting of the waves, which the norm needs too.
template <int KT, int NW>
__global__ __launch_bounds__(64 * NW, 2) void delta_blocks_kernel(RunArgs ra) {
  extern __shared__ __align__(16) float lds[];
  const zp_delta& a = ra.d;
  constexpr int NC = 2, dk = 16 * KT, dv = 32 * NW, size = block_floats(dk, dv);
  const int tid = threadIdx.x, lane = tid & 63, l16 = lane & 15, g = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  float* const red = lds + 2 * size;           // [2][NW * 16]
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
  const float* const base = ra.ws + (block_slot(ra.row0, sg, seg, 0) * a.heads + h) * size;
  const int64_t stride = (int64_t)a.heads * size;
  const int blocks = (sg.count + kBlock - 1) / kBlock;
  auto request = [&](int b) {                  // a block behind the last: nothing is read
    const StageLoads from(base + b * stride, b < blocks ? size * 4 : 0);
#pragma unroll
    for (int u = 0; u < (size / 256 + NW - 1) / NW; ++u) {
      const int i = min(wave + u * NW, size / 256 - 1);            // the last may come twice
      from.ld(lds + (b & 1) * size + i * 256, lane * 16, i * 1024);
    }
  };
  f32x4 O[NC];
  uint16_t gate[NC][4];
  const float inv_v = 1.f / (float)a.vdim;
  const int out_at = (4 * g * (int)a.out_stride + h * dv + col0 + l16) * 2;
  const int low_at = (4 * g * (int)a.low_stride + a.g_at + h * dv + col0 + l16) * 2;
  f32x4 done[NC];
  auto finish = [&](int b) {                   // rows of block b, whose squares are in red; none of block -1
    const f32x4 ss = block_squares_total<NW>(red + (b & 1) * NW * kBlock);
    const int cnt = b < 0 ? 0 : min(kBlock, sg.count - b * kBlock);
    const BlockRows out(a.out, sg.row + b * kBlock, cnt, a.out_stride);
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const float rs = __builtin_amdgcn_rsqf(ss[r] * inv_v + a.eps);
#pragma unroll
      for (int nc = 0; nc < NC; ++nc)
        out.st(out_at + r * (int)a.out_stride * 2, nc * 16, done[nc][r] * rs * nrm[nc] * fast_sigmoid(bf16_bits_to_float(gate[nc][r])));
    }
  };
  request(0);
  __builtin_amdgcn_s_waitcnt(0);               // the state is there: the loop's first use of it must not wait in every pass
#pragma unroll 1
  for (int b = 0; b < blocks; ++b) {
    wait_and_meet();
    request(b + 1);
    finish(b - 1);
    const int cnt = min(kBlock, sg.count - b * kBlock);
    const BlockRows low(a.low, sg.row + b * kBlock, cnt, a.low_stride);
#pragma unroll
    for (int r = 0; r < 4; ++r)
#pragma unroll
      for (int nc = 0; nc < NC; ++nc) gate[nc][r] = low.ld(low_at + r * (int)a.low_stride * 2, nc * 16);
    const float* const blk = lds + (b & 1) * size + lane * 4;
    f32x4 U[NC];
#pragma unroll
    for (int nc = 0; nc < NC; ++nc) {
      U[nc] = *(const f32x4*)(blk + 3 * kBlock * dk + (wave * NC + nc) * 256);
      O[nc] = f32x4{0.f, 0.f, 0.f, 0.f};
    }
#pragma unroll
    for (int kt = 0; kt < KT; ++kt) {
      const f32x4 W = *(const f32x4*)(blk + kt * 256), Q = *(const f32x4*)(blk + (KT + kt) * 256);
#pragma unroll
      for (int j = 0; j < 4; ++j)
#pragma unroll
        for (int nc = 0; nc < NC; ++nc) {
          U[nc] = mfma_f32_step(W[j], S[kt][nc][j], U[nc]);
          O[nc] = mfma_f32_step(Q[j], S[kt][nc][j], O[nc]);
        }
    }
    const f32x4 P = *(const f32x4*)(blk + kBlock * (3 * dk + dv));
    const float* const dec = blk - lane * 4 + kBlock * (3 * dk + dv) + kBlock * kBlock + 4 * g;
#pragma unroll
    for (int kt = 0; kt < KT; ++kt) {
      const f32x4 d = *(const f32x4*)(dec + 16 * kt), K = *(const f32x4*)(blk + (2 * KT + kt) * 256);
#pragma unroll
      for (int nc = 0; nc < NC; ++nc) {
        S[kt][nc] *= d;
        mfma_f32_16(K, U[nc], S[kt][nc]);
      }
    }
#pragma unroll
    for (int nc = 0; nc < NC; ++nc) mfma_f32_16(P, U[nc], O[nc]);
    block_squares<NC>(O, red + (b & 1) * NW * kBlock, wave);
#pragma unroll
    for (int nc = 0; nc < NC; ++nc) done[nc] = O[nc];
  }
  wait_and_meet();
  finish(blocks - 1);
  store_state<KT, NC>(S, state, dv, col0);
  // the last inputs of the head's convolutions (runs are longer than a filter)
  const int taps = a.taps, cw = 2 * dk + dv, hk = h / (a.heads / a.kv_heads);
  char* const tail = (char*)a.conv_state + item * (taps - 1) * cw * 2;
  for (int i = tid; i < (taps - 1) * cw; i += blockDim.x) {
    const int e = i / cw, c = i - e * cw;
    const int at = c < dk ? hk * dk + c : (c < 2 * dk ? a.kv_heads * dk + hk * dk + c - dk : 2 * a.kv_heads * dk + h * dv + c - 2 * dk);
    Elem<BF16>::st(tail, i, Elem<BF16>::ld(a.in, (int64_t)(sg.row + max(sg.count - (taps - 1) + e, 0)) * a.in_stride + at));
  }
}

template <int KT, int NW> int launch_blocks(const RunArgs& ra, hipStream_t st) {
  constexpr int smem = (2 * block_floats(16 * KT, 32 * NW) + 2 * NW * kBlock) * 4;
  if (smem > 60 * 1024 && hipFuncSetAttribute((const void*)delta_blocks_kernel<KT, NW>, hipFuncAttributeMaxDynamicSharedMemorySize,
                                              smem) != hipSuccess) {
    zp_set_error("delta_runs: cannot reserve %d bytes of LDS", smem);
    return ZP_EHIP;
  }
  hipLaunchKernelGGL((delta_blocks_kernel<KT, NW>), dim3((unsigned)((int64_t)ra.d.seg.n * ra.d.heads)), dim3(64 * NW), smem, st, ra);
  ZP_LAUNCH_CHECK();
  return ZP_OK;
}
template <int KT> int launch_blocks(const RunArgs& ra, hipStream_t st) {
  switch (ra.d.dv / 32) {
    case 1: return launch_blocks<KT, 1>(ra, st);
    case 2: return launch_blocks<KT, 2>(ra, st);
    case 3: return launch_blocks<KT, 3>(ra, st);
    default: return launch_blocks<KT, 4>(ra, st);
  }
}

template <int TAPS> int launch_prepare(const RunArgs& ra, int longest, hipStream_t st) {
  const zp_delta& a = ra.d;
  const size_t smem = sizeof(float) * (kBlock * 4 * 132 + 2 * kBlock * kBlock + kBlock);
  if (smem > 60 * 1024 && hipFuncSetAttribute((const void*)delta_prepare_kernel<TAPS>, hipFuncAttributeMaxDynamicSharedMemorySize,
                                              (int)smem) != hipSuccess) {
    zp_set_error("delta_runs: cannot reserve %zu bytes of LDS", smem);
    return ZP_EHIP;
  }
  hipLaunchKernelGGL((delta_prepare_kernel<TAPS>), dim3((unsigned)((longest + kBlock - 1) / kBlock), (unsigned)a.heads, (unsigned)a.seg.n),
                     dim3(256), smem, st, ra);
  ZP_LAUNCH_CHECK();
  return ZP_OK;
}

int launch_runs(const RunArgs& ra, int longest, hipStream_t st) {
  const zp_delta& a = ra.d;
  const int rc = a.taps <= 4 ? launch_prepare<4>(ra, longest, st) : launch_prepare<kMaxTaps>(ra, longest, st);
  if (rc != ZP_OK) return rc;
  switch (a.dk) {
    case 32: return launch_blocks<2>(ra, st);
    case 64: return launch_blocks<4>(ra, st);
    default: return launch_blocks<8>(ra, st);
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
  if (dtype != ZP_BF16 || (a.dk != 32 && a.dk != 64 && a.dk != 128) || a.dv % 32 || a.dv > 128 || a.taps < 1 || a.taps > kMaxTaps || a.heads > 65535 ||
      a.seg.n > 65535 || a.in_stride % 8 || a.low_stride % 8 || a.out_stride >= (1 << 24) || a.low_stride >= (1 << 24)) {
    zp_set_error("delta_runs: bfloat16, head sizes %d (32, 64, 128) and %d (a multiple of 32, <= 128), %d taps (1 .. %d) unsupported",
                 a.dk, a.dv, a.taps, kMaxTaps);
    return ZP_EUNSUPPORTED;
  }
  if (a.seg.n == 0 || longest == 0) return ZP_OK;
  ZP_REQUIRE(a.in && a.low && a.filters && a.a_log && a.dt_bias && a.norm && a.state && (a.conv_state || a.taps == 1) && a.out &&
                 a.seg.rows && a.seg.counts && a.seg.slots && a.seg.starts && aligned16(a.state) && aligned16(a.in) && aligned16(a.low) &&
                 aligned16(a.dt_bias) && aligned16(workspace),
             "delta_runs: null or unaligned pointer");
  ZP_REQUIRE(workspace && workspace_bytes >= zp_delta_runs_workspace(a.seg.num_rows - first_row, a.seg.n, a.heads, a.dk, a.dv),
             "delta_runs: workspace too small");
  RunArgs ra = {a, (float*)workspace, first_row};
  ra.d.seg.max_count = longest;               // no segment has more blocks than were prepared
  return launch_runs(ra, longest, (hipStream_t)stream);
}
