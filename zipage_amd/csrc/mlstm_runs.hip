// Matrix memory with exponential gates (mlstm.hip) over long runs, 16 tokens at a time.  With F_t the sum of
// the block's log forget gates up to token t, x_s = i_s - F_s and m the running maximum,
//
//   D[t, s] = e^{F_t + x_s - m_t} q_t . k_s (s <= t),  a_t = e^{F_t + m_0 - m_t}
//   O = a (Q S) + D V,   n . q_t = a_t (n . q_t) + sum_s D[t, s]
//   S <- e^{F_15 + m_0 - m_15} S + sum_s e^{F_15 + x_s - m_15} k_s v_s^T,  n likewise with k alone
//
// One workgroup per (segment, head) walks the blocks with S in registers; all fp32 (the products q . k on
// the bf16 matrix cores are exact products of the projections, added up in fp32).
#include "blocks.h"

namespace {

template <typename T, int KT, int NC>
__global__ __launch_bounds__(NC == 2 ? 256 : 512) void mlstm_blocks_kernel(zp_mlstm a) {
  extern __shared__ __align__(16) float lds[];
  __shared__ float red[2][16 * kBlock];
  constexpr int dk = 16 * KT, kKs = dk + 4;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, nw = blockDim.x >> 6, l16 = lane & 15, g = lane >> 4;
  const int dv = a.dv;
  const int h = blockIdx.x % a.heads;
  const Segment sg = segment_of(a.seg, blockIdx.x / a.heads);
  if (sg.count <= 0) return;
  float* const kl = lds;                       // [2][16][kKs] keys of the block
  float* const nl = kl + 2 * kBlock * kKs;     // [2][dk] normaliser
  float* const state = a.state + ((int64_t)sg.slot * a.heads + h) * ((int64_t)dk * dv + dk + 4);
  float* const nstate = state + (int64_t)dk * dv;
  const bool fresh = sg.start == 0;
  const int col0 = wave * 16 * NC;
  f32x4 S[KT][NC];
  load_state<KT, NC>(S, state, dv, col0, fresh);
  for (int c = tid; c < dk; c += blockDim.x) nl[c] = fresh ? 0.f : nstate[c];
  float m = fresh ? 0.f : nstate[dk];
  float nrm[NC];
#pragma unroll
  for (int nc = 0; nc < NC; ++nc) nrm[nc] = a.norm[h * dv + col0 + nc * 16 + l16] * a.out_scale;
  const float icap = 1.f / a.cap, ib = a.i_bias[h], fb = a.f_bias[h];
  const int blocks = (sg.count + kBlock - 1) / kBlock;

  // what a block reads: its token l16's gates and query, keys for the stage, values
  float zi, zf;
  f32x4 q[KT];
  float v[NC][4];
  constexpr int kPieces = kBlock * dk / 4 / 256 > 0 ? kBlock * dk / 4 / 256 : 1;
  f32x4 kp[kPieces];
  auto fetch = [&](int b) {
    const int cnt = min(kBlock, sg.count - b * kBlock);
    const int64_t row = sg.row + b * kBlock, mine = row + min(l16, cnt - 1);
    zi = a.gates[mine * a.gate_stride + h];
    zf = a.gates[mine * a.gate_stride + a.heads + h];
#pragma unroll
    for (int kt = 0; kt < KT; ++kt) q[kt] = load4<T>(a.in, mine * a.in_stride + a.q_at + h * dk + kt * 16 + 4 * g);
#pragma unroll
    for (int nc = 0; nc < NC; ++nc)
#pragma unroll
      for (int r = 0; r < 4; ++r)
        v[nc][r] = Elem<T>::ld(a.in, (row + min(4 * g + r, cnt - 1)) * a.in_stride + a.v_at + h * dv + col0 + nc * 16 + l16);
#pragma unroll
    for (int i = 0; i < kPieces; ++i) {
      const int p = tid + i * blockDim.x;
      if (p < kBlock * dk / 4) {
        const int t = p / (dk / 4), c = (p % (dk / 4)) * 4;
        kp[i] = load4<T>(a.in, (row + min(t, cnt - 1)) * a.in_stride + a.k_at + h * dk + c);
      }
    }
  };
  auto stage = [&](int buf, int b) {
    (void)b;
#pragma unroll
    for (int i = 0; i < kPieces; ++i) {
      const int p = tid + i * blockDim.x;
      if (p < kBlock * dk / 4) *(f32x4*)(kl + (buf * kBlock + p / (dk / 4)) * kKs + (p % (dk / 4)) * 4) = kp[i];
    }
    // workgroups of fewer threads than pieces: the rest straight from memory
    for (int p = tid + kPieces * blockDim.x; p < kBlock * dk / 4; p += blockDim.x) {
      const int cnt = min(kBlock, sg.count - b * kBlock), t = p / (dk / 4), c = (p % (dk / 4)) * 4;
      *(f32x4*)(kl + (buf * kBlock + t) * kKs + c) =
          load4<T>(a.in, (sg.row + b * kBlock + min(t, cnt - 1)) * a.in_stride + a.k_at + h * dk + c);
    }
  };
  fetch(0);
  stage(0, 0);
  __syncthreads();
  for (int b = 0; b < blocks; ++b) {
    const int cnt = min(kBlock, sg.count - b * kBlock), buf = b & 1;
    const int64_t row = sg.row + b * kBlock;
    float gate[NC][4];
#pragma unroll
    for (int nc = 0; nc < NC; ++nc)
#pragma unroll
      for (int r = 0; r < 4; ++r)
        gate[nc][r] = Elem<T>::ld(a.in, (row + min(4 * g + r, cnt - 1)) * a.in_stride + a.g_at + h * dv + col0 + nc * 16 + l16);
    // ---- gates of token l16
    float gi = -INFINITY, gf = 0.f;
    if (l16 < cnt) {
      gi = a.cap * tanhf((zi + ib) * icap);
      const float x = a.cap * tanhf((zf + fb) * icap);
      gf = fminf(x, 0.f) - log1pf(expf(-fabsf(x)));
    }
    const float m0 = m;
    float F = 0.f, F_all = 0.f, mt = 0.f;
#pragma unroll
    for (int t = 0; t < kBlock; ++t) {
      const float ft = __builtin_bit_cast(float, __builtin_amdgcn_readlane(__builtin_bit_cast(int, gf), t));
      const float it = __builtin_bit_cast(float, __builtin_amdgcn_readlane(__builtin_bit_cast(int, gi), t));
      m = fmaxf(ft + m, it);
      F_all += ft;
      if (l16 == t) { F = F_all; mt = m; }
    }
    const float x = gi - F;                                   // -inf behind the last token
    const float inter = expf(F + m0 - mt), keep = expf(F_all + m0 - m), wr = expf(F_all + x - m), floor_ = expf(-mt);
    // ---- q . k and its weights: rows s = 4 g + r, column t = l16
    f32x4 P = {0.f, 0.f, 0.f, 0.f};
    const float* const kb = kl + buf * kBlock * kKs;
    if constexpr (T::bytes == 2) {
      // the same bf16 values as in memory: 32 channels per product, in the order lane group g holds them
#pragma unroll
      for (int kt = 0; kt < KT; kt += 2) {
        const f32x4 k0 = *(const f32x4*)(kb + l16 * kKs + kt * 16 + 4 * g), k1 = *(const f32x4*)(kb + l16 * kKs + kt * 16 + 16 + 4 * g);
        const u32x4 kf = {pack_bf16(k0[0], k0[1]), pack_bf16(k0[2], k0[3]), pack_bf16(k1[0], k1[1]), pack_bf16(k1[2], k1[3])};
        const u32x4 qf = {pack_bf16(q[kt][0], q[kt][1]), pack_bf16(q[kt][2], q[kt][3]), pack_bf16(q[kt + 1][0], q[kt + 1][1]),
                          pack_bf16(q[kt + 1][2], q[kt + 1][3])};
        P = mfma_bf16(kf, qf, P);
      }
    } else {
#pragma unroll
      for (int kt = 0; kt < KT; ++kt) {
        const f32x4 k0 = *(const f32x4*)(kb + l16 * kKs + kt * 16 + 4 * g);
        mfma_f32_16(k0, q[kt], P);
      }
    }
    float nq = 0.f;
    const float* const nb = nl + buf * dk;
#pragma unroll
    for (int kt = 0; kt < KT; ++kt) {
      const f32x4 n4 = *(const f32x4*)(nb + kt * 16 + 4 * g);
#pragma unroll
      for (int j = 0; j < 4; ++j) nq = fmaf(q[kt][j], n4[j], nq);
    }
    nq *= inter;
    float wrow[4], irow[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int s = 4 * g + r;
      const float xs = __shfl(x, s);
      wrow[r] = __shfl(wr, s);
      irow[r] = __shfl(inter, s);
      P[r] = s <= l16 && s < cnt ? P[r] * expf(F + xs - mt) : 0.f;
      nq += P[r];
    }
    nq += lane_xor16(nq);
    nq += lane_xor32(nq);
    const float den = fmaxf(fabsf(nq) * a.q_scale, floor_) + 1e-6f;
    const float unden = 1.f / den;
    // ---- read-outs
    f32x4 O[NC];
#pragma unroll
    for (int nc = 0; nc < NC; ++nc) O[nc] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int kt = 0; kt < KT; ++kt)
#pragma unroll
      for (int j = 0; j < 4; ++j)
#pragma unroll
        for (int nc = 0; nc < NC; ++nc) O[nc] = mfma_f32_step(q[kt][j], S[kt][nc][j], O[nc]);
#pragma unroll
    for (int nc = 0; nc < NC; ++nc) {
      const f32x4 vt = {v[nc][0], v[nc][1], v[nc][2], v[nc][3]};
#pragma unroll
      for (int r = 0; r < 4; ++r) O[nc][r] *= irow[r];
      mfma_f32_16(P, vt, O[nc]);
    }
    // ---- state and normaliser behind the block
#pragma unroll
    for (int nc = 0; nc < NC; ++nc)
#pragma unroll
      for (int r = 0; r < 4; ++r) v[nc][r] *= wrow[r];
    f32x4 vw[NC];
#pragma unroll
    for (int nc = 0; nc < NC; ++nc) vw[nc] = f32x4{v[nc][0], v[nc][1], v[nc][2], v[nc][3]};
    fetch(min(b + 1, blocks - 1));
#pragma unroll
    for (int kt = 0; kt < KT; ++kt) {
      f32x4 kT;
#pragma unroll
      for (int j = 0; j < 4; ++j) kT[j] = kb[(4 * g + j) * kKs + kt * 16 + l16];
#pragma unroll
      for (int nc = 0; nc < NC; ++nc) {
        S[kt][nc] *= keep;
        mfma_f32_16(kT, vw[nc], S[kt][nc]);
      }
    }
    for (int c = tid; c < dk; c += blockDim.x) {
      float n = nb[c] * keep;
#pragma unroll
      for (int s = 0; s < kBlock; ++s)
        n = fmaf(__builtin_bit_cast(float, __builtin_amdgcn_readlane(__builtin_bit_cast(int, wr), s)), kb[s * kKs + c], n);
      nl[(buf ^ 1) * dk + c] = n;
    }
    stage(buf ^ 1, min(b + 1, blocks - 1));
    // ---- norm, gate, store
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const float f = __shfl(unden, 4 * g + r) * a.q_scale;
#pragma unroll
      for (int nc = 0; nc < NC; ++nc) O[nc][r] *= f;
    }
    block_squares<NC>(O, red[buf]);
    __syncthreads();
    const f32x4 ss = block_squares_total(red[buf], nw);
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
  for (int c = tid; c < dk; c += blockDim.x) nstate[c] = nl[(blocks & 1) * dk + c];
  if (tid == 0) nstate[dk] = m;
}

template <typename T, int KT> int launch_blocks(const zp_mlstm& a, hipStream_t st) {
  const unsigned grid = (unsigned)((int64_t)a.seg.n * a.heads);
  const size_t smem = sizeof(float) * (2 * kBlock * (16 * KT + 4) + 2 * 16 * KT);
  const bool narrow = (int64_t)grid * (a.dv / 32) < 1024;      // half the columns per wave, twice the waves
  if (narrow) hipLaunchKernelGGL((mlstm_blocks_kernel<T, KT, 1>), dim3(grid), dim3(a.dv * 4), smem, st, a);
  else hipLaunchKernelGGL((mlstm_blocks_kernel<T, KT, 2>), dim3(grid), dim3(a.dv * 2), smem, st, a);
  ZP_LAUNCH_CHECK();
  return ZP_OK;
}

}  // namespace

extern "C" int zp_mlstm_runs(const zp_mlstm* args, int32_t dtype, void* stream) {
  ZP_REQUIRE(args, "mlstm_runs: null arguments");
  const zp_mlstm& a = *args;
  ZP_REQUIRE(a.seg.n >= 0 && a.heads > 0 && a.vdim > 0 && a.vdim <= a.dv && a.cap > 0.f && a.seg.num_slots > 0 &&
                 a.gate_stride >= 2 * a.heads && a.out_stride >= (int64_t)a.heads * a.dv, "mlstm_runs: bad dims");
  ZP_MODEL_DTYPE("mlstm_runs");
  if ((a.dk != 32 && a.dk != 64 && a.dk != 128) || a.dv % 32 || a.dv > 128 || a.in_stride % 8 || a.q_at % 8 || a.k_at % 8) {
    zp_set_error("mlstm_runs: head sizes %d (32, 64, 128) and %d (a multiple of 32, <= 128) unsupported", a.dk, a.dv);
    return ZP_EUNSUPPORTED;
  }
  if (a.seg.n == 0) return ZP_OK;
  ZP_REQUIRE(a.in && a.gates && a.i_bias && a.f_bias && a.norm && a.state && a.out && a.seg.rows && a.seg.counts &&
                 a.seg.slots && a.seg.starts && aligned16(a.in) && aligned16(a.state), "mlstm_runs: null or unaligned pointer");
  hipStream_t st = (hipStream_t)stream;
#define ZP_MLSTM(T)                                    \
  switch (a.dk) {                                      \
    case 32: return launch_blocks<T, 2>(a, st);        \
    case 64: return launch_blocks<T, 4>(a, st);        \
    default: return launch_blocks<T, 8>(a, st);        \
  }
  if (dtype == ZP_BF16) { ZP_MLSTM(BF16); } else { ZP_MLSTM(F32); }
#undef ZP_MLSTM
}
