// Matrix memory with exponential gates (mlstm.hip) over long runs, 16 tokens at a time.  With F_t the sum of
// the block's log forget gates up to token t, x_s = i_s - F_s and m the running maximum,
//
//   D[t, s] = e^{F_t + x_s - m_t} q_t . k_s (s <= t),  a_t = e^{F_t + m_0 - m_t}
//   O = a (Q S) + D V,   n . q_t = a_t (n . q_t) + sum_s D[t, s]
//   S <- e^{F_15 + m_0 - m_15} S + sum_s e^{F_15 + x_s - m_15} k_s v_s^T,  n likewise with k alone
//
//   mlstm_gates     gates and the running maximum, one wave per head and sequence
//   mlstm_prepare   D and the block's factors, for all blocks at once
//   mlstm_blocks    a head's blocks one after the other, S in registers
//
// All fp32: the products q . k on the bf16 matrix cores are exact products of the projections, added up in
// fp32; those with S run on the fp32 ones.  Projections in bfloat16.
#include "blocks.h"
#include <type_traits>

namespace {

struct RunArgs {
  zp_mlstm d;
  float* aux;    // per block and head: kAux floats
  float4* scal;  // per token row from row0 on and head: F, x, m, m before the block
  int row0;
};
// D as a left operand (256), then a, write factors, e^{-m}, row sums of D (16 each), the keep factor
constexpr int kAux = 512, kInter = 256, kWrite = 272, kFloor = 288, kSum = 304, kKeep = 320;

__device__ __forceinline__ float lane_value(float v, int lane) {
  return __builtin_bit_cast(float, __builtin_amdgcn_readlane(__builtin_bit_cast(int, v), lane));
}

// lane i <- lane i - N of its row of 16, or `edge`
template <int N> __device__ __forceinline__ float row_shr(float v, float edge) {
  return __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(__builtin_bit_cast(int, edge), __builtin_bit_cast(int, v), 0x110 + N,
                                                               0xf, 0xf, false));
}

__global__ __launch_bounds__(64) void mlstm_gates_kernel(RunArgs ra) {
  const zp_mlstm& a = ra.d;
  const int lane = threadIdx.x, h = blockIdx.x % a.heads;
  const Segment sg = segment_of(a.seg, blockIdx.x / a.heads);
  if (sg.count <= 0 || sg.row < ra.row0) return;
  float* const mstate = a.state + ((int64_t)sg.slot * a.heads + h) * ((int64_t)a.dk * a.dv + a.dk + 4) + (int64_t)a.dk * a.dv + a.dk;
  float m = sg.start == 0 ? 0.f : *mstate;
  const float icap = 1.f / a.cap, ib = a.i_bias[h], fb = a.f_bias[h];
  float zi = 0.f, zf = 0.f;
  auto fetch = [&](int t0) {
    const int64_t src = (int64_t)(sg.row + min(t0 + lane, sg.count - 1)) * a.gate_stride + h;
    zi = a.gates[src];
    zf = a.gates[src + a.heads];
  };
  fetch(0);
  for (int t0 = 0; t0 < sg.count; t0 += 64) {
    const int cnt = min(64, sg.count - t0);
    const float gi = a.cap * tanhf((zi + ib) * icap), x = a.cap * tanhf((zf + fb) * icap);
    const float gf = fminf(x, 0.f) - log1pf(expf(-fabsf(x)));
    fetch(t0 + 64);
    // sums and maxima inside each block of 16 lanes: m_t = F_t + max(m before the block, max_{s <= t} x_s)
    float F = lane < cnt ? gf : 0.f;
    F += row_shr<1>(F, 0.f);
    F += row_shr<2>(F, 0.f);
    F += row_shr<4>(F, 0.f);
    F += row_shr<8>(F, 0.f);
    const float xs = lane < cnt ? gi - F : -INFINITY;
    float top = xs;
    top = fmaxf(top, row_shr<1>(top, -INFINITY));
    top = fmaxf(top, row_shr<2>(top, -INFINITY));
    top = fmaxf(top, row_shr<4>(top, -INFINITY));
    top = fmaxf(top, row_shr<8>(top, -INFINITY));
    float m0 = m;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      if (lane >> 4 == r) m0 = m;
      m = lane_value(F, r * 16 + 15) + fmaxf(m, lane_value(top, r * 16 + 15));     // rows behind the end change nothing
    }
    const float mine_m = F + fmaxf(m0, top);
    if (lane < cnt)
      ra.scal[(int64_t)(sg.row + t0 + lane - ra.row0) * a.heads + h] = make_float4(F, xs, mine_m, m0);
  }
  if (lane == 0) *mstate = m;
}

// A wave per (block, head).
template <int KT>
__global__ __launch_bounds__(256) void mlstm_prepare_kernel(RunArgs ra) {
  const zp_mlstm& a = ra.d;
  const int lane = threadIdx.x & 63, l16 = lane & 15, g = lane >> 4, h = blockIdx.y * 4 + (threadIdx.x >> 6);
  const Segment sg = segment_of(a.seg, blockIdx.z);
  const int t0 = blockIdx.x * kBlock;
  if (t0 >= sg.count || sg.row < ra.row0 || h >= a.heads) return;
  const int cnt = min(kBlock, sg.count - t0);
  const int64_t mine = sg.row + t0 + min(l16, cnt - 1);
  const float4 sc = ra.scal[(mine - ra.row0) * a.heads + h];
  const uint16_t* const in = (const uint16_t*)a.in + mine * a.in_stride + h * (16 * KT) + g * 8;
  f32x4 P = {0.f, 0.f, 0.f, 0.f};              // rows s = 4 g + r, column t = l16
#pragma unroll
  for (int ks = 0; ks < KT / 2; ++ks)
    P = mfma_bf16(*(const u32x4*)(in + a.k_at + ks * 32), *(const u32x4*)(in + a.q_at + ks * 32), P);
  float sum = 0.f;
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int s = 4 * g + r;
    const float xs = __shfl(sc.y, s);
    P[r] = s <= l16 && s < cnt && l16 < cnt ? P[r] * expf(sc.x + xs - sc.z) : 0.f;
    sum += P[r];
  }
  sum += lane_xor16(sum);
  sum += lane_xor32(sum);
  const float F_end = lane_value(sc.x, cnt - 1), m_end = lane_value(sc.z, cnt - 1);
  float* const aux = ra.aux + (block_slot(ra.row0, sg, blockIdx.z, blockIdx.x) * a.heads + h) * kAux;
  *(f32x4*)(aux + lane * 4) = P;
  if (g == 0) {
    aux[kInter + l16] = expf(sc.x + sc.w - sc.z);
    aux[kWrite + l16] = l16 < cnt ? expf(F_end + sc.y - m_end) : 0.f;
    aux[kFloor + l16] = expf(-sc.z);
    aux[kSum + l16] = sum;
    if (l16 == 0) aux[kKeep] = expf(F_end + sc.w - m_end);
  }
}

// LDS of a stage: Q and K rows, their 16-byte pieces xor-ed with the row so that neither operand order meets
// bank conflicts; V rows; the block's factors.  The next stage comes in while this one is worked on.
template <int KT, int NW>
__global__ __launch_bounds__(64 * NW, 2) void mlstm_blocks_kernel(RunArgs ra) {
  extern __shared__ __align__(16) char lds_raw[];
  const zp_mlstm& a = ra.d;
  constexpr int NC = 2, dk = 16 * KT, dv = 32 * NW, PR = dk / 8;     // PR: pieces per row of Q and K
  const int tid = threadIdx.x, lane = tid & 63, l16 = lane & 15, g = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int h = blockIdx.x % a.heads, seg = blockIdx.x / a.heads;
  const Segment sg = segment_of(a.seg, seg);
  if (sg.count <= 0 || sg.row < ra.row0) return;
  constexpr int v_bytes = kBlock * dv * 2, stage = 2 * kBlock * dk * 2 + v_bytes + kAux * 4;
  float (*const red)[NW * kBlock] = (float (*)[NW * kBlock])(lds_raw + 2 * stage);
  float (*const den)[kBlock] = (float (*)[kBlock])(red + 2);
  float (*const nl)[dk] = (float (*)[dk])(den + 2);
  float* const state = a.state + ((int64_t)sg.slot * a.heads + h) * ((int64_t)dk * dv + dk + 4);
  float* const nstate = state + (int64_t)dk * dv;
  const bool fresh = sg.start == 0;
  const int col0 = wave * 16 * NC;
  f32x4 S[KT][NC];
  load_state<KT, NC>(S, state, dv, col0, fresh);
  for (int c = tid; c < dk; c += blockDim.x) nl[0][c] = fresh ? 0.f : nstate[c];
  float nrm[NC];
#pragma unroll
  for (int nc = 0; nc < NC; ++nc) nrm[nc] = a.norm[h * dv + col0 + nc * 16 + l16] * a.out_scale;
  const int blocks = (sg.count + kBlock - 1) / kBlock;
  const float* const aux0 = ra.aux + (block_slot(ra.row0, sg, seg, 0) * a.heads + h) * kAux;
  constexpr int kQK = KT / 2;                  // KBs of Q, and of K
  // a share of `kbs` KBs; the last may come twice
  auto share = [&](auto kbs, auto ld) {
#pragma unroll
    for (int u = 0; u < (kbs.value + NW - 1) / NW; ++u) ld(min(wave + u * NW, kbs.value - 1));
  };
  auto request = [&](int b) {                  // of a block behind the last nothing is read
    char* const st = lds_raw + (b & 1) * stage;
    const int cnt = b < blocks ? min(kBlock, sg.count - b * kBlock) : 0;
    const StageLoads rows((const char*)a.in + (int64_t)(sg.row + b * kBlock) * a.in_stride * 2, cnt * a.in_stride * 2);
    const StageLoads aux(aux0 + (int64_t)b * a.heads * kAux, cnt > 0 ? kAux * 4 : 0);
    share(std::integral_constant<int, kQK>(), [&](int i) {
      const int s = i * 64 + lane, row = s / PR, pc = (s % PR) ^ (row & (PR - 1));
      const int at = max(min(row, cnt - 1), 0) * (int)a.in_stride * 2 + pc * 16;
      rows.ld(st + i * 1024, at, (a.q_at + h * dk) * 2);
      rows.ld(st + (kQK + i) * 1024, at, (a.k_at + h * dk) * 2);
    });
    share(std::integral_constant<int, NW>(), [&](int i) {
      const int s = i * 64 + lane, row = s / (dv / 8), pc = s - row * (dv / 8);
      rows.ld(st + (2 * kQK + i) * 1024, max(min(row, cnt - 1), 0) * (int)a.in_stride * 2 + pc * 16, (a.v_at + h * dv) * 2);
    });
    share(std::integral_constant<int, 2>(), [&](int i) { aux.ld(st + (2 * kQK + NW + i) * 1024, lane * 16, i * 1024); });
  };
  f32x4 done[NC];
  f32x4 O[NC];
  uint16_t gate[NC][4];
  const float inv_v = 1.f / (float)a.vdim;
  const int out_at = (4 * g * (int)a.out_stride + h * dv + col0 + l16) * 2;
  const int gate_at = (4 * g * (int)a.in_stride + a.g_at + h * dv + col0 + l16) * 2;
  auto finish = [&](int b) {                   // rows of block b, whose squares and denominators are in LDS; none of block -1
    const f32x4 ss = block_squares_total<NW>(red[b & 1]);
    const f32x4 dn = *(const f32x4*)(den[b & 1] + 4 * g);
    const int cnt = b < 0 ? 0 : min(kBlock, sg.count - b * kBlock);
    const BlockRows out(a.out, sg.row + b * kBlock, cnt, a.out_stride);
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const float f = a.q_scale * __builtin_amdgcn_rcpf(dn[r]), rs = f * __builtin_amdgcn_rsqf(ss[r] * f * f * inv_v + a.eps);
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
    const BlockRows gp(a.in, sg.row + b * kBlock, cnt, a.in_stride);
#pragma unroll
    for (int r = 0; r < 4; ++r)
#pragma unroll
      for (int nc = 0; nc < NC; ++nc) gate[nc][r] = gp.ld(gate_at + r * (int)a.in_stride * 2, nc * 16);
    const char* const st = lds_raw + (b & 1) * stage;
    const char* const ks = st + kBlock * dk * 2;
    const uint16_t* const vs = (const uint16_t*)(ks + kBlock * dk * 2);
    const float* const aux = (const float*)((const char*)vs + v_bytes);
    // ---- read-outs
#pragma unroll
    for (int nc = 0; nc < NC; ++nc) O[nc] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int kt = 0; kt < KT; ++kt) {
      const f32x4 q = load4<BF16>(st + l16 * dk * 2 + (((2 * kt + (g >> 1)) ^ (l16 & (PR - 1))) * 16) + (g & 1) * 8, 0);
#pragma unroll
      for (int j = 0; j < 4; ++j)
#pragma unroll
        for (int nc = 0; nc < NC; ++nc) O[nc] = mfma_f32_step(q[j], S[kt][nc][j], O[nc]);
    }
    const f32x4 P = *(const f32x4*)(aux + lane * 4), inter = *(const f32x4*)(aux + kInter + 4 * g), wr = *(const f32x4*)(aux + kWrite + 4 * g);
    const float keep = aux[kKeep];
    f32x4 v[NC];
#pragma unroll
    for (int nc = 0; nc < NC; ++nc) {
      v[nc] = read_columns((const char*)(vs + (4 * g + (l16 >> 2)) * dv + col0 + nc * 16 + (l16 & 3) * 4));
      O[nc] *= inter;
      mfma_f32_16(P, v[nc], O[nc]);
      v[nc] *= wr;
    }
    // ---- the state behind the block
    const int kr = 4 * g + (l16 >> 2), kz = ((l16 & 3) >> 1) ^ (kr & (PR - 1));
    const char* const krow = ks + kr * dk * 2 + (l16 & 1) * 8;
#pragma unroll
    for (int kt = 0; kt < KT; ++kt) {
      const f32x4 kT = read_columns(krow + (((2 * kt) ^ kz) * 16));
#pragma unroll
      for (int nc = 0; nc < NC; ++nc) {
        S[kt][nc] *= keep;
        mfma_f32_16(kT, v[nc], S[kt][nc]);
      }
    }
    block_squares<NC>(O, red[b & 1], wave);
#pragma unroll
    for (int nc = 0; nc < NC; ++nc) done[nc] = O[nc];
    // ---- the normaliser: 16 lanes a token
    const float* const n = nl[b & 1];
#pragma unroll
    for (int u = 0; u < (kBlock + 4 * NW - 1) / (4 * NW); ++u) {
      const int t = min((tid >> 4) + u * 4 * NW, kBlock - 1), pc = min(l16, PR - 1);
      float q[8], d = 0.f;
      Vec8<BF16>::ld(st + t * dk * 2 + ((pc ^ (t & (PR - 1))) * 16), 0, q);
#pragma unroll
      for (int i = 0; i < 8; ++i) d = fmaf(q[i], n[pc * 8 + i], d);
      d = row16_sum(l16 < PR ? d : 0.f);
      const float x = fmaxf(fabsf(fmaf(aux[kInter + t], d, aux[kSum + t])) * a.q_scale, aux[kFloor + t]) + 1e-6f;
      if (l16 == 0) den[b & 1][t] = x;
    }
#pragma unroll
    for (int u = 0; u < (KT + 4 * NW - 1) / (4 * NW); ++u) {
      const int kt = min(wave * 4 + g + u * 4 * NW, KT - 1);         // channel 16 kt + l16
      float x = n[kt * 16 + l16] * keep;
#pragma unroll
      for (int s4 = 0; s4 < 4; ++s4) {
        const int r = 4 * s4 + (l16 >> 2);
        const f32x4 k4 = read_columns(ks + r * dk * 2 + (((2 * kt + ((l16 & 3) >> 1)) ^ (r & (PR - 1))) * 16) + (l16 & 1) * 8);
        const f32x4 w4 = *(const f32x4*)(aux + kWrite + 4 * s4);
#pragma unroll
        for (int i = 0; i < 4; ++i) x = fmaf(w4[i], k4[i], x);
      }
      nl[(b + 1) & 1][kt * 16 + l16] = x;
    }
  }
  wait_and_meet();
  finish(blocks - 1);
  store_state<KT, NC>(S, state, dv, col0);
  for (int c = tid; c < dk; c += blockDim.x) nstate[c] = nl[blocks & 1][c];
}

template <int KT, int NW> int launch_blocks(const RunArgs& ra, hipStream_t st) {
  constexpr int dk = 16 * KT, dv = 32 * NW;
  constexpr size_t smem = 2 * (2 * kBlock * dk * 2 + kBlock * dv * 2 + kAux * 4) + 2 * 4 * (NW * kBlock + kBlock + dk);
  hipLaunchKernelGGL((mlstm_blocks_kernel<KT, NW>), dim3((unsigned)((int64_t)ra.d.seg.n * ra.d.heads)), dim3(64 * NW), smem, st, ra);
  ZP_LAUNCH_CHECK();
  return ZP_OK;
}

template <int KT> int launch_runs(const RunArgs& ra, int longest, hipStream_t st) {
  const zp_mlstm& a = ra.d;
  const unsigned grid = (unsigned)((int64_t)a.seg.n * a.heads);
  hipLaunchKernelGGL(mlstm_gates_kernel, dim3(grid), dim3(64), 0, st, ra);
  hipLaunchKernelGGL((mlstm_prepare_kernel<KT>), dim3((unsigned)((longest + kBlock - 1) / kBlock), (unsigned)((a.heads + 3) / 4), (unsigned)a.seg.n),
                     dim3(256), 0, st, ra);
  ZP_LAUNCH_CHECK();
  switch (a.dv / 32) {
    case 1: return launch_blocks<KT, 1>(ra, st);
    case 2: return launch_blocks<KT, 2>(ra, st);
    case 3: return launch_blocks<KT, 3>(ra, st);
    default: return launch_blocks<KT, 4>(ra, st);
  }
}

}  // namespace

extern "C" int64_t zp_mlstm_runs_workspace(int32_t rows, int32_t segments, int32_t heads) {
  if (rows < 0 || segments < 0 || heads <= 0) return -1;
  return (((int64_t)rows / kBlock + segments) * kAux + (int64_t)rows * 4) * heads * 4;
}

extern "C" int zp_mlstm_runs(const zp_mlstm* args, int32_t first_row, int32_t longest, void* workspace,
                             int64_t workspace_bytes, int32_t dtype, void* stream) {
  ZP_REQUIRE(args, "mlstm_runs: null arguments");
  const zp_mlstm& a = *args;
  ZP_REQUIRE(a.seg.n >= 0 && a.heads > 0 && a.vdim > 0 && a.vdim <= a.dv && a.cap > 0.f && a.seg.num_slots > 0 &&
                 a.gate_stride >= 2 * a.heads && a.out_stride >= (int64_t)a.heads * a.dv && first_row >= 0 && longest >= 0 &&
                 first_row <= a.seg.num_rows, "mlstm_runs: bad dims");
  if (dtype != ZP_BF16 || (a.dk != 32 && a.dk != 64 && a.dk != 128) || a.dv % 32 || a.dv > 128 || a.in_stride % 8 || a.q_at % 8 ||
      a.k_at % 8 || a.v_at % 8 || a.in_stride >= (1 << 24) || a.out_stride >= (1 << 24) || a.heads > 65535 || a.seg.n > 65535) {
    zp_set_error("mlstm_runs: bfloat16, head sizes %d (32, 64, 128) and %d (a multiple of 32, <= 128) unsupported", a.dk, a.dv);
    return ZP_EUNSUPPORTED;
  }
  if (a.seg.n == 0 || longest == 0) return ZP_OK;
  ZP_REQUIRE(a.in && a.gates && a.i_bias && a.f_bias && a.norm && a.state && a.out && a.seg.rows && a.seg.counts &&
                 a.seg.slots && a.seg.starts && aligned16(a.in) && aligned16(a.state) && aligned16(workspace),
             "mlstm_runs: null or unaligned pointer");
  ZP_REQUIRE(workspace && workspace_bytes >= zp_mlstm_runs_workspace(a.seg.num_rows - first_row, a.seg.n, a.heads),
             "mlstm_runs: workspace too small");
  RunArgs ra = {a, (float*)workspace, nullptr, first_row};
  ra.scal = (float4*)(ra.aux + ((int64_t)(a.seg.num_rows - first_row) / kBlock + a.seg.n) * a.heads * kAux);
  ra.d.seg.max_count = longest;               // no segment has more blocks than were prepared
  hipStream_t st = (hipStream_t)stream;
  switch (a.dk) {
    case 32: return launch_runs<2>(ra, longest, st);
    case 64: return launch_runs<4>(ra, longest, st);
    default: return launch_runs<8>(ra, longest, st);
  }
}
