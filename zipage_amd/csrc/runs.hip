// Attention of runs of prompt tokens, and the gather of the cached rows they look back on.
#include "mfma.h"

namespace {

// ------------------------------------------------------------------ gather of cached rows
__global__ __launch_bounds__(256) void gather_rows_kernel(const char* src, const int32_t* rows, char* out,
                                                          int64_t total, int pieces, int64_t num_rows) {
  const int64_t id = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (id >= total) return;
  const int64_t r = id / pieces, pc = id - r * pieces;
  int64_t s = rows[r];
  if (s < 0 || s >= num_rows) s = 0;
  ((u32x4*)out)[id] = ((const u32x4*)src)[s * pieces + pc];
}

// ------------------------------------------------------------------ runs of prompt tokens
struct TilesArgs {
  const uint16_t* q;      // token rows of q_st elements, head h at h * maps * (D + P)
  const uint16_t* k;      // key rows of kv_st elements, head h at h * maps * D
  const uint16_t* v;      // value rows of kv_st elements, head h at h * V
  const uint16_t* ks;     // rows of s_st elements: the last P of every head's key; null: P = 0
  uint16_t* out;          // token rows of o_st elements, head h at h * V
  const int32_t* tiles;   // (T, 4): first query row, queries, first key row of the run, position
                          // of the first query counted from that key
  const float* sinks;     // (H,) logits that only join the denominator, or null
  int T, H, HK, D, P, V;  // HK key / value heads; query head h uses head h / (H / HK)
  int window, chunk;      // at most one is set, see first_seen
  int64_t q_rows, k_rows, q_st, kv_st, s_st, o_st;
  float scale, out_scale;
  float cap;              // > 0: soft cap of the scores
  // two maps: rms(o1 - balance * o2) * out_scale * sigmoid(gate), the mean over vdim
  float balance, eps;
  int vdim;
  const uint16_t* gate;   // token rows of g_st elements, head h at h * V; or null
  int64_t g_st;
  const float2* turns;    // one map: (q_rows, V / 2) cos and sin, results turn back by them; or null
};

constexpr int kTileQ = 128;   // queries per workgroup
constexpr int kTileK = 64;    // keys per LDS tile

// A workgroup owns up to 128 queries of one head; key and value tiles pass through LDS once for all of
// them (double-buffered, the next tile's loads in flight during the products), a wave owns 16 * kQT
// queries at a time and skips the 32-key steps none of them sees.
// First key position a query sees: the last `window` up to and including its own, or those of its own
// block of `chunk` positions (key 0 of the run starts a block), or all.
__device__ __forceinline__ int first_seen(int pos, int window, int chunk) {
  if (window > 0) return max(0, pos - window + 1);
  return chunk > 0 ? pos / chunk * chunk : 0;
}

// Two maps: one workgroup of eight waves per CU; else two of four waves, which share its 160 KB.
constexpr int tile_waves(int maps) { return maps == 2 ? 8 : 4; }

template <int DKS, int VCB, int MAPS> struct TileStage {
  static constexpr int kK = MAPS * DKS * 32 + 8, kV = VCB * 128 + 8;    // row strides: rows 16 bytes apart in the banks
  static constexpr int kElems = kTileK * (kK + kV);
  static constexpr int kWaves = tile_waves(MAPS);
  static constexpr int kBuffers = MAPS == 2 || 8 * kElems <= 160 * 1024 ? 2 : 1;
  static constexpr int kBytes = kBuffers * kElems * 2;
};

enum { kNoCap, kCap, kBoundedCap };   // of the scores, see SoftCap

// Column tile t of a wave: 16 queries, map t % MAPS of the head (differential attention has two, over the same
// values; elsewhere there is one).  SHARED: the last P elements of every head's key are the row of a.ks.
template <int DKS, int VCB, int kQT, int MAPS, bool SHARED, int CAP>
__global__ __launch_bounds__(64 * tile_waves(MAPS), 2) void run_tiles_kernel(TilesArgs a) {
  extern __shared__ __align__(16) char lds_raw[];
  typedef TileStage<DKS, VCB, MAPS> Stage;
  constexpr bool kTurns = MAPS == 1 && !SHARED && CAP == kNoCap;
  constexpr int kT = kQT * MAPS, kWaves = Stage::kWaves, kThreads = 64 * kWaves, kPass = 16 * kQT * kWaves;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l16 = lane & 15, g = lane >> 4;
  const int h = blockIdx.x % a.H, tile = blockIdx.x / a.H;   // one head's tiles share an L2 when H % 8 == 0
  const int q0 = a.tiles[tile * 4], nq = min(a.tiles[tile * 4 + 1], kTileQ);
  const int kb = a.tiles[tile * 4 + 2], rel = a.tiles[tile * 4 + 3];
  // host-made descriptors: rows outside the buffers are not touched
  if (q0 < 0 || kb < 0 || rel < 0 || (int64_t)q0 + nq > a.q_rows || (int64_t)kb + rel + nq > a.k_rows) return;
  const int DT = a.D + (SHARED ? a.P : 0);
  const SoftCap cap(a.scale, a.cap);
  const int hk = h / (a.H / a.HK);
  const uint16_t* kbase = a.k + (int64_t)kb * a.kv_st + hk * MAPS * a.D;
  const uint16_t* vbase = a.v + (int64_t)kb * a.kv_st + hk * a.V;
  const uint16_t* sbase = SHARED ? a.ks + (int64_t)kb * a.s_st : nullptr;

  for (int wg0 = 0; wg0 < nq; wg0 += kPass) {                 // uniform in the workgroup
    const int w0 = wg0 + wave * 16 * kQT;
    const int last = rel + min(wg0 + kPass, nq) - 1;          // last key any query of the pass sees
    const int first = first_seen(rel + wg0, a.window, a.chunk);
    const int hi = w0 < nq ? rel + min(w0 + 16 * kQT, nq) - 1 : -1;      // the same for the wave
    const int lo = first_seen(rel + w0, a.window, a.chunk);
    const int lo_last = first_seen(rel + w0 + 16 * kQT - 1, a.window, a.chunk);

    u32x4 qf[kT][DKS];
    int qpos[kQT], qlow[kQT];                                 // keys qlow .. qpos are seen
#pragma unroll
    for (int t = 0; t < kT; ++t) {
      const int qi = min(w0 + t / MAPS * 16 + l16, nq - 1);
      qpos[t / MAPS] = rel + qi;
      qlow[t / MAPS] = first_seen(rel + qi, a.window, a.chunk);
      const uint16_t* q = a.q + (int64_t)(q0 + qi) * a.q_st + (h * MAPS + t % MAPS) * DT;
#pragma unroll
      for (int ks = 0; ks < DKS; ++ks) {
        // past the head's end: the key columns there hold other elements, against zeros here
        const int c = ks * 32 + g * 8;
        qf[t][ks] = *(const u32x4*)(q + (c < DT ? c : 0));
        if (c >= DT) qf[t][ks] = u32x4{0u, 0u, 0u, 0u};
      }
    }
    f32x4 o[kT][VCB * 8];
    float m[kT], l[kT];
#pragma unroll
    for (int t = 0; t < kT; ++t) {
      m[t] = CAP == kBoundedCap ? 0.f : -INFINITY;
      l[t] = 0.f;
#pragma unroll
      for (int i = 0; i < VCB * 8; ++i) o[t][i] = f32x4{0.f, 0.f, 0.f, 0.f};
    }

    constexpr int kKP = 4 * MAPS * DKS, kVP = 16 * VCB;        // pieces of a key row, DKS * 4 per map, and of a value row
    constexpr int kKN = kTileK * kKP / kThreads, kVN = kTileK * kVP / kThreads;
    u32x4 rk[kKN], rv[kVN];                                    // this thread's pieces of a tile
    auto fetch = [&](int k0) {                                 // offsets from the tile's first row: 32 bits
      const uint16_t *kt = kbase + k0 * a.kv_st, *vt = vbase + k0 * a.kv_st, *st = SHARED ? sbase + k0 * a.s_st : nullptr;
      const uint32_t kv_st = (uint32_t)a.kv_st, s_st = (uint32_t)a.s_st;
#pragma unroll
      for (int j = 0; j < kKN; ++j) {
        const int id = tid + kThreads * j, pc = id % kKP, map = pc / (4 * DKS), c = (pc % (4 * DKS)) * 8;
        const uint32_t r = min(id / kKP, last - k0);
        if (SHARED) {
          const bool own = c < a.D;
          rk[j] = *(const u32x4*)((own ? kt : st) + (own ? r * kv_st + c : r * s_st + (c < DT ? c - a.D : 0)));
        } else {
          rk[j] = *(const u32x4*)(kt + (r * kv_st + map * a.D + (c < a.D ? c : 0)));
        }
      }
#pragma unroll
      for (int j = 0; j < kVN; ++j) {
        const int id = tid + kThreads * j, c = (id % kVP) * 8;
        const uint32_t r = min(id / kVP, last - k0);
        rv[j] = *(const u32x4*)(vt + (r * kv_st + (c < a.V ? c : 0)));
      }
    };
    fetch(first);
    if (Stage::kBuffers == 2) __syncthreads();                 // a pass before this one still reads its tiles
    int buf = 0;
    for (int t0 = first; t0 <= last; t0 += kTileK, buf ^= 1) {
      if (Stage::kBuffers == 1) __syncthreads();               // the tile before this one is used up
      uint16_t* const ldsk = (uint16_t*)lds_raw + (Stage::kBuffers == 2 ? buf * Stage::kElems : 0);
      uint16_t* const ldsv = ldsk + kTileK * Stage::kK;
#pragma unroll
      for (int j = 0; j < kKN; ++j) {
        const int id = tid + kThreads * j;
        *(u32x4*)(ldsk + id / kKP * Stage::kK + (id % kKP) * 8) = rk[j];
      }
#pragma unroll
      for (int j = 0; j < kVN; ++j) {
        const int id = tid + kThreads * j;
        *(u32x4*)(ldsv + id / kVP * Stage::kV + (id % kVP) * 8) = rv[j];
      }
      __syncthreads();
      if (t0 + kTileK <= last) fetch(t0 + kTileK);
#pragma unroll 1
      for (int sub = 0; sub < kTileK; sub += 32) {
        const int k0 = t0 + sub;
        if (k0 > hi || k0 + 31 < lo) continue;                 // uniform in the wave
        f32x4 s[kT][2];
#pragma unroll
        for (int tt = 0; tt < 2; ++tt) {
#pragma unroll
          for (int t = 0; t < kT; ++t) s[t][tt] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
          for (int ks = 0; ks < DKS; ++ks)
#pragma unroll
            for (int map = 0; map < MAPS; ++map) {
              const u32x4 kf = *(const u32x4*)(ldsk + (sub + tt * 16 + l16) * Stage::kK + (map * DKS + ks) * 32 + g * 8);
#pragma unroll
              for (int t = map; t < kT; t += MAPS) s[t][tt] = mfma_bf16(kf, qf[t][ks], s[t][tt]);
            }
        }
        // every query of the wave sees all 32 keys: no masks
        const bool inner = k0 + 31 <= rel + w0 && k0 >= lo_last;
        u32x4 pf[kT];
#pragma unroll
        for (int t = 0; t < kT; ++t) {
          float p[8], sum = 0.f;
#pragma unroll
          for (int i = 0; i < 8; ++i) {
            const float x = s[t][i >> 2][i & 3];
            p[i] = CAP == kNoCap ? x * cap.factor : cap.capped(x);
          }
          if (!inner) {
#pragma unroll
            for (int i = 0; i < 8; ++i) {
              const int key = k0 + step_key(g, i);
              if (key > qpos[t / MAPS] || key < qlow[t / MAPS]) p[i] = -INFINITY;
            }
          }
          float ms = 0.f, f = 1.f;
          if (CAP != kBoundedCap) {
            float mx = -INFINITY;
#pragma unroll
            for (int i = 0; i < 8; ++i) mx = fmaxf(mx, p[i]);
            mx = fmaxf(mx, lane_xor16(mx));
            mx = fmaxf(mx, lane_xor32(mx));
            const float mn = fmaxf(m[t], mx);
            ms = mn == -INFINITY ? 0.f : mn;                    // a query whose window starts later
            f = __builtin_amdgcn_exp2f(m[t] - ms);
            m[t] = mn;
          }
#pragma unroll
          for (int i = 0; i < 8; ++i) {
            p[i] = __builtin_amdgcn_exp2f(CAP == kBoundedCap ? p[i] : p[i] - ms);
            sum += p[i];
          }
          l[t] = CAP == kBoundedCap ? l[t] + sum : l[t] * f + sum;
          if (CAP != kBoundedCap && __any(f != 1.f)) {
#pragma unroll
            for (int i = 0; i < VCB * 8; ++i) o[t][i] *= f;
          }
          pf[t] = u32x4{pack_bf16(p[0], p[1]), pack_bf16(p[2], p[3]), pack_bf16(p[4], p[5]),
                        pack_bf16(p[6], p[7])};
        }
#pragma unroll
        for (int cb = 0; cb < VCB; ++cb) {
          u32x4 v[8];
#pragma unroll
          for (int i = 0; i < 8; ++i)
            v[i] = *(const u32x4*)(ldsv + (sub + step_key(g, i)) * Stage::kV + cb * 128 + l16 * 8);
#pragma unroll
          for (int c = 0; c < 8; ++c) {
            const u32x4 vf = column_of(v, c);
#pragma unroll
            for (int t = 0; t < kT; ++t) o[t][cb * 8 + c] = mfma_bf16(vf, pf[t], o[t][cb * 8 + c]);
          }
        }
      }
    }
#pragma unroll
    for (int qt = 0; qt < kQT; ++qt) {
      float inv[MAPS];
#pragma unroll
      for (int map = 0; map < MAPS; ++map) {
        float lt = l[qt * MAPS + map];
        lt += lane_xor16(lt);
        lt += lane_xor32(lt);
        if (MAPS == 1 && a.sinks) lt += __builtin_amdgcn_exp2f(a.sinks[h] * 1.44269504088896f - m[qt]);
        inv[map] = lt > 0.f ? 1.f / lt : 0.f;
      }
      if constexpr (MAPS == 1) {
        inv[0] *= a.out_scale;
      } else {                                                 // o1 <- rms(o1 / l1 - balance * o2 / l2) * out_scale
        const float second = a.balance * inv[1];
        float ss = 0.f;
#pragma unroll
        for (int j = 0; j < VCB * 8; ++j)
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            const float r = o[qt * 2][j][i] * inv[0] - o[qt * 2 + 1][j][i] * second;
            o[qt * 2][j][i] = r;
            if ((j >> 3) * 128 + (4 * g + i) * 8 < a.V) ss += r * r;
          }
        ss += lane_xor16(ss);
        ss += lane_xor32(ss);
        inv[0] = a.out_scale / sqrtf(ss / (float)a.vdim + a.eps);
      }
      const int qi = w0 + qt * 16 + l16;
      if (qi >= nq) continue;
      uint16_t* out = a.out + (int64_t)(q0 + qi) * a.o_st + h * a.V;
      const float2* turns = a.turns;
      asm volatile("" : "+s"(turns));                          // nothing of the way back is computed before the loop
      const uint16_t* gate = MAPS == 2 && a.gate ? a.gate + (int64_t)(q0 + qi) * a.g_st + h * a.V : nullptr;
#pragma unroll
      for (int cb = 0; cb < VCB; ++cb)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int col = cb * 128 + (4 * g + i) * 8;
          if (col < a.V) {
            float r[8];
#pragma unroll
            for (int c = 0; c < 8; ++c) r[c] = o[qt * MAPS][cb * 8 + c][i] * inv[0];
            if (kTurns && turns) turn_back8(r, turns + ((int64_t)(q0 + qi) * a.V + col) / 2);
            if (MAPS == 2 && gate) {
              float z[8];
              Vec8<BF16>::ld(gate, col, z);
#pragma unroll
              for (int c = 0; c < 8; ++c) r[c] *= sigmoid_of<BF16>(z[c]);
            }
            Vec8<BF16>::st(out, col, r);
          }
        }
    }
  }
}

template <int DKS, int VCB, int kQT, int MAPS, bool SHARED, int CAP> int launch_run_tiles(const TilesArgs& a, hipStream_t st) {
  constexpr int smem = TileStage<DKS, VCB, MAPS>::kBytes;
  if (smem > 64 * 1024 &&
      hipFuncSetAttribute((const void*)run_tiles_kernel<DKS, VCB, kQT, MAPS, SHARED, CAP>,
                          hipFuncAttributeMaxDynamicSharedMemorySize, smem) != hipSuccess) {
    zp_set_error("run_attention: cannot reserve %d bytes of LDS", smem);
    return ZP_EHIP;
  }
  hipLaunchKernelGGL((run_tiles_kernel<DKS, VCB, kQT, MAPS, SHARED, CAP>), dim3((unsigned)a.T * a.H),
                     dim3(64 * TileStage<DKS, VCB, MAPS>::kWaves), smem, st, a);
  ZP_LAUNCH_CHECK();
  return ZP_OK;
}

template <bool SHARED, int CAP> int launch_one_map(const TilesArgs& a, hipStream_t st) {
  const int dk = (a.D + a.P + 31) / 32;
  if (a.V <= 128) {
    if (dk <= 2) return launch_run_tiles<2, 1, 2, 1, SHARED, CAP>(a, st);
    if (dk <= 4) return launch_run_tiles<4, 1, 2, 1, SHARED, CAP>(a, st);
    if (dk <= 6) return launch_run_tiles<6, 1, 2, 1, SHARED, CAP>(a, st);
    return launch_run_tiles<8, 1, 2, 1, SHARED, CAP>(a, st);
  }
  if (dk <= 4) return launch_run_tiles<4, 2, 1, 1, SHARED, CAP>(a, st);
  return launch_run_tiles<8, 2, 1, 1, SHARED, CAP>(a, st);
}
template <int CAP> int launch_two_maps(const TilesArgs& a, hipStream_t st) {
  const int dk = (a.D + 31) / 32;
  if (a.V <= 128) {
    if (dk <= 2) return launch_run_tiles<2, 1, 1, 2, false, CAP>(a, st);
    return launch_run_tiles<4, 1, 1, 2, false, CAP>(a, st);
  }
  return launch_run_tiles<4, 2, 1, 2, false, CAP>(a, st);
}
template <int CAP> int launch_forms(const TilesArgs& a, bool two, hipStream_t st) {
  return two ? launch_two_maps<CAP>(a, st) : launch_one_map<false, CAP>(a, st);
}

}  // namespace

extern "C" int zp_gather_rows(const void* src, const int32_t* rows, void* out, int32_t n,
                              int32_t row_bytes, int64_t num_rows, void* stream) {
  ZP_REQUIRE(n >= 0 && row_bytes > 0 && row_bytes % 16 == 0 && num_rows > 0, "gather_rows: bad dims");
  if (n == 0) return ZP_OK;
  ZP_REQUIRE(src && rows && out && aligned16(src) && aligned16(out), "gather_rows: null or unaligned pointer");
  const int pieces = row_bytes / 16;
  const int64_t total = (int64_t)n * pieces;
  hipLaunchKernelGGL(gather_rows_kernel, dim3((unsigned)((total + 255) / 256)), dim3(256), 0,
                     (hipStream_t)stream, (const char*)src, rows, (char*)out, total, pieces, num_rows);
  ZP_LAUNCH_CHECK();
  return ZP_OK;
}

extern "C" int zp_run_attention(const void* q, const void* k, const void* v, const void* k_shared, void* out,
                                const int32_t* tiles, const float* sinks, const zp_attention_form* form, int32_t T,
                                int32_t H, int32_t HK, int32_t D, int32_t P, int32_t V, int32_t window,
                                int32_t chunk, int64_t q_rows, int64_t k_rows, int64_t q_stride,
                                int64_t kv_stride, int64_t shared_stride, int64_t out_stride, float scale,
                                float out_scale, int32_t dtype, void* stream) {
  const zp_attention_form plain = {0.f, 1, 0.f, 0.f, 0, nullptr, 0, nullptr}, f = form ? *form : plain;
  const bool two = f.maps == 2;
  ZP_REQUIRE(T >= 0 && H > 0 && HK > 0 && H % HK == 0 && D > 0 && P >= 0 && V > 0 && window >= 0 && chunk >= 0 &&
                 !(window && chunk) && (f.maps == 1 || two) && f.softcap >= 0.f && (P > 0) == (k_shared != nullptr),
             "run_attention: bad dims");
  if (dtype != ZP_BF16 || D % 8 != 0 || P % 8 != 0 || D + P > (two ? 128 : 256) || V % 8 != 0 || V > 256) {
    zp_set_error("run_attention: bfloat16, D %d + %d (multiples of 8, <= 256, of two maps <= 128), V %d (multiple of 8, <= 256)",
                 D, P, V);
    return ZP_EUNSUPPORTED;
  }
  if (T == 0) return ZP_OK;
  ZP_REQUIRE(q && k && v && out && tiles, "run_attention: null pointer");
  ZP_REQUIRE(!P || f.softcap == 0.f, "run_attention: shared keys go without a soft cap");
  ZP_REQUIRE(!f.turns || (!P && f.softcap == 0.f && aligned16(f.turns)), "run_attention: turns go without shared keys and soft cap");
  ZP_REQUIRE(!two || (!sinks && !P && !f.turns && f.vdim > 0 && f.vdim <= V && (!f.gate || f.gate_stride >= (int64_t)H * V)),
             "run_attention: two maps go without sinks, shared keys and turns, with a mean over the values");
  ZP_REQUIRE(aligned16(q) && aligned16(k) && aligned16(v) && aligned16(out) && aligned16(k_shared) && aligned16(f.gate) &&
                 f.gate_stride % 8 == 0 && q_stride % 8 == 0 && kv_stride % 8 == 0 && shared_stride % 8 == 0 &&
                 out_stride % 8 == 0 && q_stride >= (int64_t)H * f.maps * (D + P) && out_stride >= (int64_t)H * V &&
                 (!P || shared_stride >= P) && (int64_t)T * H < (1ll << 31) &&
                 kv_stride < (1ll << 26) && shared_stride < (1ll << 26),
             "run_attention: unaligned rows or too many tiles");
  TilesArgs a = {(const uint16_t*)q, (const uint16_t*)k, (const uint16_t*)v, (const uint16_t*)k_shared, (uint16_t*)out,
                 tiles, sinks, T, H, HK, D, P, V, window, chunk, q_rows, k_rows, q_stride, kv_stride, shared_stride,
                 out_stride, scale, out_scale, f.softcap, f.balance, f.eps, f.vdim, (const uint16_t*)f.gate, f.gate_stride,
                 (const float2*)f.turns};
  hipStream_t st = (hipStream_t)stream;
  if (P) return launch_one_map<true, kNoCap>(a, st);
  if (!(f.softcap > 0.f)) return launch_forms<kNoCap>(a, two, st);
  return soft_cap_bounded(f.softcap) ? launch_forms<kBoundedCap>(a, two, st) : launch_forms<kCap>(a, two, st);
}
