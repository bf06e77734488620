// Linear attention with decay (linear.hip) over long runs, 16 tokens at a time.  With G_t the product of the
// block's decays up to token t, per key channel, a block is
//
//   P[t, s] = sum_c q_t k_s G_t / G_s (s <= t),   O = (G q) S + P V,   S <- G_15 S + sum_s (G_15 / G_s) k_s v_s^T
//
// linear_prepare turns q and k, takes the decays, and computes everything without S for all blocks at once, in
// the order of the matrix operands; ratios of decays are running products of the decays themselves, so nothing
// is divided and nothing overflows.  linear_blocks walks a head's blocks with S in registers.  All fp32;
// projections in bfloat16.
#include "blocks.h"
#include "linear.h"
#include <type_traits>

namespace {

struct RunArgs {
  zp_linear d;
  float* ws;
  int row0;      // first token row of the first segment
};

// G q and the keys as left operands, P, the block's decays; whole KBs
__host__ __device__ inline constexpr int block_floats(int dk) {
  return (2 * kBlock * dk + kBlock * kBlock + dk + 255) / 256 * 256;
}

__global__ __launch_bounds__(256, 4) void linear_prepare_kernel(RunArgs ra) {
  const zp_linear& a = ra.d;
  constexpr int ld = 132;                      // every row: reads across tokens meet no conflicts, offsets are constants
  __shared__ __align__(16) float qs[kBlock * ld], ks[kBlock * ld], gs[kBlock * ld], Ps[kBlock * kBlock];
  const int dk = a.dk, half = a.rot / 2;
  const Segment sg = segment_of(a.seg, blockIdx.z);
  const int t0 = blockIdx.x * kBlock;
  if (t0 >= sg.count || sg.row < ra.row0) return;
  const int cnt = min(kBlock, sg.count - t0);
  const int h = blockIdx.y;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const float fixed = a.low ? 1.f : a.decay[h];
#pragma unroll
  for (int u = 0; u < 2; ++u) {                // dk <= 128: two pieces a thread at most
    const int i = tid + u * 256, t = i / (dk / 4), c = (i - t * (dk / 4)) * 4;
    if (t >= kBlock) continue;
    f32x4 q = {0.f, 0.f, 0.f, 0.f}, k = q, g = {1.f, 1.f, 1.f, 1.f};
    if (t < cnt) {
      const int64_t row = sg.row + t0 + t;
      q = load4<BF16>(a.in, row * a.in_stride + a.q_at + h * dk + c) * a.q_scale;
      k = load4<BF16>(a.in, row * a.in_stride + a.k_at + h * dk + c) * a.k_scale;
      g *= fixed;
      if (a.low) {
        const f32x4 z = load4<BF16>(a.low, row * a.low_stride + h * dk + c) + *(const f32x4*)(a.decay + h * dk + c);
#pragma unroll
        for (int e = 0; e < 4; ++e) g[e] = __expf(-a.inv_tau * fast_softplus(-z[e]));
      }
    }
    *(f32x4*)(qs + t * ld + c) = q;
    *(f32x4*)(ks + t * ld + c) = k;
    *(f32x4*)(gs + t * ld + c) = g;
  }
  __syncthreads();
  if (half > 0) {                              // uniform
    for (int i = tid; i < cnt * half; i += 256) {
      const int t = i / half, c = i - t * half;
      const float2 r = rotary_turn(sg.start + t0 + t, a.freqs[c]);
      float* const q = qs + t * ld + c;
      float* const k = ks + t * ld + c;
      turn_pair(q[0], q[half], r.x, r.y);
      turn_pair(k[0], k[half], r.x, r.y);
    }
    __syncthreads();
  }
  // ---- P: 16 lanes walk k_s down the tokens, in pieces of four channels; group i of wave w takes s = w + 4 i
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
      f32x4 pp = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int p = 0; p < 2; ++p) {
        const f32x4 gt = *(const f32x4*)(gs + t * ld + at[p]);
#pragma unroll
        for (int e = 0; e < 4; ++e) kk[p][e] *= t > s ? gt[e] : 1.f;
        pp += kk[p] * *(const f32x4*)(qs + t * ld + at[p]);
      }
      const float sp = row16_sum((pp[0] + pp[1]) + (pp[2] + pp[3]));
      Ps[t * kBlock + s] = t >= s ? sp : 0.f;                  // all 16 lanes, the same value
      if (t % 4 == 3) __builtin_amdgcn_sched_barrier(0);       // not all tokens' rows in registers at once
    }
  }
  __syncthreads();
  // ---- columns: a thread reads and writes its own only
  float* const oQ = ra.ws + (block_slot(ra.row0, sg, blockIdx.z, blockIdx.x) * a.heads + h) * block_floats(dk);
  float* const oK = oQ + kBlock * dk;          // [dk / 16][64 lanes][4], as oQ
  float* const oP = oK + kBlock * dk;          // [64][4]
  float* const oG = oP + kBlock * kBlock;      // [dk]
  if (tid < dk) {                              // G q
    const int c = tid;
    float G = 1.f;
#pragma unroll
    for (int t = 0; t < kBlock; ++t) {
      G *= gs[t * ld + c];
      qs[t * ld + c] *= G;
    }
    oG[c] = G;
  }
  if (tid >= 256 - dk) {                       // keys, on the threads the queries leave free as far as they go
    const int c = tid - (256 - dk);
    float R = 1.f;
#pragma unroll
    for (int g = 3; g >= 0; --g) {
      f32x4 x;
#pragma unroll
      for (int r = 3; r >= 0; --r) {
        const int t = 4 * g + r;
        x[r] = ks[t * ld + c] * R;
        R *= gs[t * ld + c];
      }
      *(f32x4*)(oK + ((c >> 4) * 64 + g * 16 + (c & 15)) * 4) = x;
    }
  }
  __syncthreads();
  if (tid < 64) *(f32x4*)(oP + tid * 4) = *(const f32x4*)(Ps + (tid & 15) * kBlock + (tid >> 4) * 4);
  for (int i = tid; i < kBlock * dk / 4; i += 256) {           // lane (g, row) of tile kt: columns 16 kt + 4 g ..
    const int l = i & 63, kt = i >> 6;
    *(f32x4*)(oQ + i * 4) = *(const f32x4*)(qs + (l & 15) * ld + kt * 16 + (l >> 4) * 4);
  }
}

// A head's blocks, one after the other: a block's operands and value rows come straight into LDS while the block
// before it is worked on; its rows are normed and stored behind the next meeting of the waves, which the norm
// needs too.
template <int KT, int NW>
__global__ __launch_bounds__(64 * NW, 2) void linear_blocks_kernel(RunArgs ra) {
  extern __shared__ __align__(16) float lds[];
  const zp_linear& a = ra.d;
  constexpr int NC = 2, dk = 16 * KT, dv = 32 * NW, size = block_floats(dk), stage = size + kBlock * dv / 2;
  const int tid = threadIdx.x, lane = tid & 63, l16 = lane & 15, g = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  float* const red = lds + 2 * stage;          // [2][NW * 16]
  const int h = blockIdx.x % a.heads, seg = blockIdx.x / a.heads;
  const Segment sg = segment_of(a.seg, seg);
  if (sg.count <= 0 || sg.row < ra.row0) return;
  float* const state = a.state + ((int64_t)sg.slot * a.heads + h) * ((int64_t)dk * dv);
  const int col0 = wave * 16 * NC;
  f32x4 S[KT][NC];
  load_state<KT, NC>(S, state, dv, col0, sg.start == 0);
  float nrm[NC];
#pragma unroll
  for (int nc = 0; nc < NC; ++nc) nrm[nc] = a.norm[h * dv + col0 + nc * 16 + l16];
  const float* const base = ra.ws + (block_slot(ra.row0, sg, seg, 0) * a.heads + h) * size;
  const int64_t stride = (int64_t)a.heads * size;
  const int blocks = (sg.count + kBlock - 1) / kBlock;
  auto request = [&](int b) {                  // a block behind the last: nothing is read
    float* const st = lds + (b & 1) * stage;
    const int cnt = b < blocks ? min(kBlock, sg.count - b * kBlock) : 0;
    const StageLoads from(base + b * stride, cnt > 0 ? size * 4 : 0);
#pragma unroll
    for (int u = 0; u < (size / 256 + NW - 1) / NW; ++u) {
      const int i = min(wave + u * NW, size / 256 - 1);            // the last may come twice
      from.ld(st + i * 256, lane * 16, i * 1024);
    }
    const StageLoads rows((const char*)a.in + (int64_t)(sg.row + b * kBlock) * a.in_stride * 2, cnt * a.in_stride * 2);
    const int s = wave * 64 + lane, row = s / (dv / 8), pc = s - row * (dv / 8);
    rows.ld(st + size + wave * 256, max(min(row, cnt - 1), 0) * (int)a.in_stride * 2 + pc * 16, (a.v_at + h * dv) * 2);
  };
  f32x4 O[NC], done[NC];
  uint16_t gate[NC][4];
  const float inv_v = 1.f / (float)a.vdim;
  const int out_at = (4 * g * (int)a.out_stride + h * dv + col0 + l16) * 2;
  const int gate_at = (4 * g * (int)a.in_stride + a.g_at + h * dv + col0 + l16) * 2;
  auto finish = [&](int b) {                   // rows of block b, whose squares are in red; none of block -1
    const f32x4 ss = block_squares_total<NW>(red + (b & 1) * NW * kBlock);
    const int cnt = b < 0 ? 0 : min(kBlock, sg.count - b * kBlock);
    const BlockRows out(a.out, sg.row + b * kBlock, cnt, a.out_stride);
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const float rs = __builtin_amdgcn_rsqf(ss[r] * inv_v + a.eps);
#pragma unroll
      for (int nc = 0; nc < NC; ++nc) {
        const float z = bf16_bits_to_float(gate[nc][r]);
        out.st(out_at + r * (int)a.out_stride * 2, nc * 16, done[nc][r] * rs * nrm[nc] * z * fast_sigmoid(z));
      }
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
    const BlockRows gp(a.in, sg.row + b * kBlock, cnt, a.in_stride);
#pragma unroll
    for (int r = 0; r < 4; ++r)
#pragma unroll
      for (int nc = 0; nc < NC; ++nc) gate[nc][r] = gp.ld(gate_at + r * (int)a.in_stride * 2, nc * 16);
    const float* const blk = lds + (b & 1) * stage + lane * 4;
    const uint16_t* const vs = (const uint16_t*)(lds + (b & 1) * stage + size);
    f32x4 v[NC];
#pragma unroll
    for (int nc = 0; nc < NC; ++nc) {
      v[nc] = read_columns((const char*)(vs + (4 * g + (l16 >> 2)) * dv + col0 + nc * 16 + (l16 & 3) * 4));
      O[nc] = f32x4{0.f, 0.f, 0.f, 0.f};
    }
#pragma unroll
    for (int kt = 0; kt < KT; ++kt) {
      const f32x4 Q = *(const f32x4*)(blk + kt * 256);
#pragma unroll
      for (int j = 0; j < 4; ++j)
#pragma unroll
        for (int nc = 0; nc < NC; ++nc) O[nc] = mfma_f32_step(Q[j], S[kt][nc][j], O[nc]);
    }
    const f32x4 P = *(const f32x4*)(blk + 2 * kBlock * dk);
#pragma unroll
    for (int nc = 0; nc < NC; ++nc) mfma_f32_16(P, v[nc], O[nc]);
    const float* const dec = blk - lane * 4 + 2 * kBlock * dk + kBlock * kBlock + 4 * g;
#pragma unroll
    for (int kt = 0; kt < KT; ++kt) {
      const f32x4 d = *(const f32x4*)(dec + 16 * kt), K = *(const f32x4*)(blk + (KT + kt) * 256);
#pragma unroll
      for (int nc = 0; nc < NC; ++nc) {
        S[kt][nc] *= d;
        mfma_f32_16(K, v[nc], S[kt][nc]);
      }
    }
    block_squares<NC>(O, red + (b & 1) * NW * kBlock, wave);
#pragma unroll
    for (int nc = 0; nc < NC; ++nc) done[nc] = O[nc];
  }
  wait_and_meet();
  finish(blocks - 1);
  store_state<KT, NC>(S, state, dv, col0);
}

template <int KT, int NW> int launch_blocks(const RunArgs& ra, hipStream_t st) {
  constexpr int smem = (2 * (block_floats(16 * KT) + kBlock * 16 * NW) + 2 * NW * kBlock) * 4;
  static_assert(smem <= 60 * 1024, "a stage outgrew the default LDS limit");
  hipLaunchKernelGGL((linear_blocks_kernel<KT, NW>), dim3((unsigned)((int64_t)ra.d.seg.n * ra.d.heads)), dim3(64 * NW), smem, st, ra);
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

}  // namespace

extern "C" int64_t zp_linear_runs_workspace(int32_t rows, int32_t segments, int32_t heads, int32_t dk) {
  if (rows < 0 || segments < 0 || heads <= 0 || dk <= 0) return -1;
  return ((int64_t)rows / kBlock + segments) * heads * block_floats(dk) * 4;
}

extern "C" int zp_linear_runs(const zp_linear* args, int32_t first_row, int32_t longest, void* workspace,
                              int64_t workspace_bytes, int32_t dtype, void* stream) {
  ZP_REQUIRE(args, "linear_runs: null arguments");
  const zp_linear& a = *args;
  ZP_REQUIRE(linear_dims_fit(a) && first_row >= 0 && longest >= 0 && first_row <= a.seg.num_rows, "linear_runs: bad dims");
  if (dtype != ZP_BF16 || (a.dk != 32 && a.dk != 64 && a.dk != 128) || a.dv % 32 || a.dv > 128 || a.heads > 65535 ||
      a.seg.n > 65535 || a.in_stride % 8 || a.q_at % 8 || a.k_at % 8 || a.v_at % 8 || a.low_stride % 8 ||
      a.in_stride >= (1 << 24) || a.out_stride >= (1 << 24)) {
    zp_set_error("linear_runs: bfloat16, head sizes %d (32, 64, 128) and %d (a multiple of 32, <= 128) unsupported", a.dk, a.dv);
    return ZP_EUNSUPPORTED;
  }
  if (a.seg.n == 0 || longest == 0) return ZP_OK;
  ZP_REQUIRE(a.in && a.decay && (a.rot == 0 || a.freqs) && a.norm && a.state && a.out && a.seg.rows && a.seg.counts &&
                 a.seg.slots && a.seg.starts && aligned16(a.in) && aligned16(a.low) && (!a.low || aligned16(a.decay)) &&
                 aligned16(a.state) && aligned16(workspace), "linear_runs: null or unaligned pointer");
  ZP_REQUIRE(workspace && workspace_bytes >= zp_linear_runs_workspace(a.seg.num_rows - first_row, a.seg.n, a.heads, a.dk),
             "linear_runs: workspace too small");
  RunArgs ra = {a, (float*)workspace, first_row};
  ra.d.seg.max_count = longest;               // no segment has more blocks than were prepared
  hipStream_t st = (hipStream_t)stream;
  hipLaunchKernelGGL(linear_prepare_kernel, dim3((unsigned)((longest + kBlock - 1) / kBlock), (unsigned)a.heads, (unsigned)a.seg.n),
                     dim3(256), 0, st, ra);
  ZP_LAUNCH_CHECK();
  switch (a.dk) {
    case 32: return launch_blocks<2>(ra, st);
    case 64: return launch_blocks<4>(ra, st);
    default: return launch_blocks<8>(ra, st);
  }
}
