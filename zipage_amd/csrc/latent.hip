// Latent attention: keys and values of all heads are linear images of one cached vector c per token
// (R elements), so the cache holds c alone, or c and a rotated key part (P elements) that all heads share.
//
//   latent_norm_store   RMS norms of the two low-rank projections of a token; c, and the key part turned by
//                       the token's position, go to its slot
//   headwise            per-head product out[n, h] = W[h] in[n, h]  (q -> W_uk^T q, sum p c -> W_uv sum p c);
//                       a tail behind each head's part passes beside it, turned
//   rotate_heads        rotary positions on a part of every head, in place
//   latent_rows         attention of single tokens over the paged latents, all heads of a token on
//                       one read of its context: score = (W_uk^T q) . c + turned q . turned k, out = sum p c
//   latent_plain        float32 form of latent_rows (true fp32 products), any sizes
//
// The attention of runs of prompt tokens over expanded keys and values is in runs.hip.
//
// The bf16 attention kernels keep S^T = K Q^T and O^T = V^T P^T: in that orientation the MFMA
// result layout of S^T (column = query, four consecutive keys per lane) IS the operand layout of
// P^T once the 32 keys of a step are numbered (lane group g holds keys 4g..4g+3 and
// 16+4g..16+4g+3), so the softmax weights never leave their lane: no LDS and no barrier in the key
// loop, every wave is its own flash loop.  V^T operands are built from row-major 16-byte loads of
// eight keys x eight columns by v_perm; the column order that results (MFMA t, row m <-> column
// 8m + t) leaves eight consecutive output columns in each lane.
#include "mfma.h"
#include <math.h>

namespace {

// ------------------------------------------------------------------ norms of the low-rank rows
struct NormStoreArgs {
  const void* in;        // (n, q_width + c_width + p_width) T
  const float* wq;       // (q_width,)
  const float* wc;       // (c_width,)
  void* q_out;           // (n, q_width) T
  void* c_out;           // (n, c_width + p_width) T or null
  void* cache;           // (num_slots, c_width + p_width) T
  const int32_t* slots;  // (n,), -1 skips
  const int32_t* positions;
  const float* freqs;    // (half,)
  int n, q_width, c_width, p_width, q_norm, c_norm, half;   // half: rotated pairs of the last part
  int64_t num_slots;
  float eps;
};
constexpr int kNormPieces = 8;   // 8-element pieces per lane: ranks up to 4096

// One wave per (token, part); without a second part, per token.
template <typename T>
__global__ __launch_bounds__(256) void latent_norm_store_kernel(NormStoreArgs a) {
  const int lane = threadIdx.x & 63;
  const int item = blockIdx.x * 4 + (threadIdx.x >> 6);
  const int row = a.c_width ? item >> 1 : item;
  if (row >= a.n) return;
  const bool is_c = a.c_width && (item & 1);
  const int width = is_c ? a.c_width : a.q_width, held = a.c_width + a.p_width;
  const int pieces = width / 8;
  const int64_t src = (int64_t)row * (a.q_width + held) + (is_c ? a.q_width : 0);
  const float* w = is_c ? a.wc : a.wq;
  float v[kNormPieces][8];
  float ss = 0.f;
#pragma unroll
  for (int k = 0; k < kNormPieces; ++k) {
    const int pc = lane + k * 64;
    if (pc < pieces) {
      Vec8<T>::ld(a.in, src + pc * 8, v[k]);
#pragma unroll
      for (int i = 0; i < 8; ++i) ss += v[k][i] * v[k][i];
    }
  }
  ss = wave_sum(ss);
  const float rs = 1.f / sqrtf(ss / (float)(is_c ? a.c_norm : a.q_norm) + a.eps);
  int64_t slot = is_c ? a.slots[row] : -1;
  if (slot >= a.num_slots) slot = -1;
#pragma unroll
  for (int k = 0; k < kNormPieces; ++k) {
    const int pc = lane + k * 64;
    if (pc < pieces) {
      float wv[8];
      Vec8<F32>::ld(w, pc * 8, wv);
#pragma unroll
      for (int i = 0; i < 8; ++i) v[k][i] = v[k][i] * rs * wv[i];
      if (is_c) {
        if (slot >= 0) Vec8<T>::st(a.cache, slot * held + pc * 8, v[k]);
        if (a.c_out) Vec8<T>::st(a.c_out, (int64_t)row * held + pc * 8, v[k]);
      } else {
        Vec8<T>::st(a.q_out, (int64_t)row * width + pc * 8, v[k]);
      }
    }
  }
  if (!is_c) return;
  // the key part: pairs (i, half + i) turn, what follows them passes
  const int rest = a.p_width - 2 * a.half;
  for (int i = lane; i < a.half + rest; i += 64) {
    float x[2];
    int at[2] = {i, i + a.half};
    const int cnt = i < a.half ? 2 : 1;
    if (cnt == 1) at[0] = i + a.half;
    for (int k = 0; k < cnt; ++k) x[k] = Elem<T>::ld(a.in, src + width + at[k]);
    if (cnt == 2) {
      const float2 r = rotary_turn(a.positions[row], a.freqs[i]);
      const float u = x[0], w2 = x[1];
      x[0] = u * r.x - w2 * r.y;
      x[1] = w2 * r.x + u * r.y;
    }
    for (int k = 0; k < cnt; ++k) {
      if (slot >= 0) Elem<T>::st(a.cache, slot * held + width + at[k], x[k]);
      if (a.c_out) Elem<T>::st(a.c_out, (int64_t)row * held + width + at[k], x[k]);
    }
  }
}

// ------------------------------------------------------------------ rotary positions in place
struct RotateArgs {
  void* x;                  // token rows of x_st elements; head h's part at h * head + at
  const int32_t* positions;
  const float* freqs;
  int n, H, head, at, half;
  int64_t x_st;
};
constexpr int kRotTokens = 4;

template <typename T, int VEC>
__global__ __launch_bounds__(256) void rotate_heads_kernel(RotateArgs a) {
  extern __shared__ __align__(16) char lds_raw[];
  float2* cs = (float2*)lds_raw;            // [kRotTokens][half]
  const int n0 = blockIdx.x * kRotTokens;
  for (int i = threadIdx.x; i < kRotTokens * a.half; i += 256) {
    const int tok = i / a.half;
    if (n0 + tok < a.n) cs[i] = rotary_turn(a.positions[n0 + tok], a.freqs[i - tok * a.half]);
  }
  __syncthreads();
  const int per_head = a.half / VEC, items = a.H * per_head;
  for (int id = threadIdx.x; id < kRotTokens * items; id += 256) {
    const int tok = id / items, it = id - tok * items;
    if (n0 + tok >= a.n) break;
    const int h = it / per_head, p = (it - h * per_head) * VEC;
    const int64_t at = (n0 + tok) * a.x_st + (int64_t)h * a.head + a.at + p;
    float u[VEC], v[VEC];
    if constexpr (VEC == 8) { Vec8<T>::ld(a.x, at, u); Vec8<T>::ld(a.x, at + a.half, v); }
    else { u[0] = Elem<T>::ld(a.x, at); v[0] = Elem<T>::ld(a.x, at + a.half); }
#pragma unroll
    for (int i = 0; i < VEC; ++i) {
      const float2 r = cs[tok * a.half + p + i];
      const float x = u[i], y = v[i];
      u[i] = x * r.x - y * r.y;
      v[i] = y * r.x + x * r.y;
    }
    if constexpr (VEC == 8) { Vec8<T>::st(a.x, at, u); Vec8<T>::st(a.x, at + a.half, v); }
    else { Elem<T>::st(a.x, at, u[0]); Elem<T>::st(a.x, at + a.half, v[0]); }
  }
}

// ------------------------------------------------------------------ per-head product
struct HeadArgs {
  const void* in;   // (n, H, K + tail) T
  const void* w;    // (H, M, K) T
  void* out;        // (n, H, M + tail) T
  const int32_t* positions;
  const float* freqs;
  int n, H, K, M, tail, half;   // behind each head's part `tail` elements, of which 2 * half turn
};

// A wave owns 16 outputs of one head for 16 * kTokTiles tokens: W is the row operand, so a lane ends
// with four consecutive outputs of one token.  Token rows past the end repeat the last one.
template <typename T, int kTokTiles>
__global__ __launch_bounds__(256) void headwise_kernel(HeadArgs a) {
  const int lane = threadIdx.x & 63, l16 = lane & 15, g = lane >> 4;
  const int m0 = (blockIdx.x * 4 + (threadIdx.x >> 6)) * 16;
  const int h = blockIdx.y;
  const int n0 = blockIdx.z * 16 * kTokTiles;
  if (a.tail && blockIdx.x == 0) {
    const int rest = a.tail - a.half;             // items of a token: the pairs, then what follows them
    for (int it = threadIdx.x; it < 16 * kTokTiles * rest; it += 256) {
      const int tok = it / rest, i = it - tok * rest, n = n0 + tok;
      if (n >= a.n) break;
      const int64_t from = ((int64_t)n * a.H + h) * (a.K + a.tail) + a.K, to = ((int64_t)n * a.H + h) * (a.M + a.tail) + a.M;
      if (i < a.half) {
        const float2 r = rotary_turn(a.positions[n], a.freqs[i]);
        const float u = Elem<T>::ld(a.in, from + i), v = Elem<T>::ld(a.in, from + i + a.half);
        Elem<T>::st(a.out, to + i, u * r.x - v * r.y);
        Elem<T>::st(a.out, to + i + a.half, v * r.x + u * r.y);
      } else {
        Elem<T>::st(a.out, to + i + a.half, Elem<T>::ld(a.in, from + i + a.half));
      }
    }
  }
  if (m0 >= a.M) return;
  f32x4 acc[kTokTiles];
#pragma unroll
  for (int t = 0; t < kTokTiles; ++t) acc[t] = f32x4{0.f, 0.f, 0.f, 0.f};
  const int64_t wrow = ((int64_t)h * a.M + m0 + l16) * a.K;
  int64_t xrow[kTokTiles];
#pragma unroll
  for (int t = 0; t < kTokTiles; ++t)
    xrow[t] = ((int64_t)min(n0 + t * 16 + l16, a.n - 1) * a.H + h) * (a.K + a.tail);
  if constexpr (T::bytes == 2) {
    const uint16_t* w = (const uint16_t*)a.w;
    const uint16_t* x = (const uint16_t*)a.in;
    const int steps = a.K / 32;
#pragma unroll 4
    for (int ks = 0; ks < steps; ++ks) {
      const int k = ks * 32 + g * 8;
      const u32x4 wf = *(const u32x4*)(w + wrow + k);
#pragma unroll
      for (int t = 0; t < kTokTiles; ++t) acc[t] = mfma_bf16(wf, *(const u32x4*)(x + xrow[t] + k), acc[t]);
    }
  } else {
    const float* w = (const float*)a.w;
    const float* x = (const float*)a.in;
    const int steps = a.K / 4;
#pragma unroll 4
    for (int ks = 0; ks < steps; ++ks) {
      const int k = ks * 4 + g;
      const float wf = w[wrow + k];
#pragma unroll
      for (int t = 0; t < kTokTiles; ++t)
        acc[t] = __builtin_amdgcn_mfma_f32_16x16x4f32(wf, x[xrow[t] + k], acc[t], 0, 0, 0);
    }
  }
#pragma unroll
  for (int t = 0; t < kTokTiles; ++t) {
    const int n = n0 + t * 16 + l16;
    if (n < a.n) {
      const int64_t at = ((int64_t)n * a.H + h) * (a.M + a.tail) + m0 + g * 4;
      if constexpr (T::bytes == 2) {
        uint2 o;
        o.x = pack_bf16(acc[t][0], acc[t][1]);
        o.y = pack_bf16(acc[t][2], acc[t][3]);
        *(uint2*)((uint16_t*)a.out + at) = o;
      } else {
        *(f32x4*)((float*)a.out + at) = acc[t];
      }
    }
  }
}

// ------------------------------------------------------------------ single tokens over the pages
struct RowsArgs {
  const void* q;          // (n, H, R + P) T
  const void* cache;      // (pages, BS, R + P) T
  const int32_t* table;   // (B, NB) page ids
  const int32_t* ctx;     // (n,) tokens of the sequence up to and including this one; 0 = inert
  const int32_t* seq;     // (n,) row of table, or null: row i
  void* out;              // (n, H, R) T
  float* part;            // splits > 1: (n, H, splits, R) fp32, then (n, H, splits, 2) max and sum
  int n, H, R, P, BS, bs_shift, B, NB, num_pages;   // P: elements that only join the scores
  int window;             // a token sees the last `window` tokens including itself; 0 = all
  int splits;             // key ranges handled by different workgroups
  int hw;                 // waves of a workgroup on different heads (1, 2, 4); the others split keys
  int lds_pages;          // page ids held in LDS
  float scale;
};

__device__ __forceinline__ int page_of(const RowsArgs& a, int t) {
  return a.bs_shift >= 0 ? t >> a.bs_shift : t / a.BS;
}

// NCB column blocks of 128 cover R.  Workgroup: one token, 16 * HT * hw heads, one key range.  A wave
// computes HT tiles of 16 heads on the same keys: with two, the second tile costs no key or value read.
//
// A wave takes 32 keys at a time.  They come from memory once, as whole 256-byte row pieces (lane: 8
// keys x 8 columns), and stay in registers as the value operand; the key operand (lane: one key, 8
// columns per MFMA) would touch 16 cache lines per 16 lanes if it were read from memory, so the wave
// passes each half of the block through an LDS stage of its own.  The next block's pieces are
// requested as the value products free their registers.  No barrier until the waves meet at the end.
// The rotated part (PK MFMA steps) is a key only, never a value: it is read as a key operand straight from
// memory, P elements of a key per four lanes.
template <int NCB, int PK> struct RowsLds {
  static constexpr int kStride = NCB * 128 + 8;                  // elements: rows 16 bytes apart in the banks
  static constexpr int kStage = 16 * kStride * 2;                // bytes per wave: 16 keys
  static constexpr int kQStride = kStride + PK * 32;             // with 64 more: an odd number of 16 bytes still
  static constexpr int kQ = 16 * kQStride * 2;                   // bytes per 16 heads
};
__host__ __device__ inline int rows_merge_floats(int R) { return 16 * (R + 4) + 32; }   // per wave

template <int NCB, int HT, int PK>
__global__ __launch_bounds__(256, NCB * HT <= 2 ? 2 : 1) void latent_rows_kernel(RowsArgs a) {
  extern __shared__ __align__(16) char lds_raw[];
  typedef RowsLds<NCB, PK> Lds;
  int* pg = (int*)lds_raw;
  char* const shared = lds_raw + ((a.lds_pages * 4 + 15) & ~15);
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int l16 = lane & 15, g = lane >> 4;
  const int hw = a.hw, kw = 4 / hw, hwi = wave % hw, kwi = wave / hw;
  uint16_t* const stage = (uint16_t*)(shared + wave * Lds::kStage);
  uint16_t* const qlds = (uint16_t*)(shared + 4 * Lds::kStage);
  const int hgroups = (a.H + 16 * HT * hw - 1) / (16 * HT * hw);
  int id = blockIdx.x;
  const int split = id % a.splits;
  id /= a.splits;
  const int hg = id % hgroups;
  const int row = id / hgroups;
  const int head0 = hg * hw * HT * 16;
  // queries to LDS, zeros past R and past the last head
  const int RW = a.R + a.P;
  constexpr int kQPieces = NCB * 16 + PK * 4;
  for (int it = tid; it < hw * HT * 16 * kQPieces; it += 256) {
    const int hl = it / kQPieces, c = (it % kQPieces) * 8;
    const int p = c - NCB * 128;                                 // >= 0: of the rotated part
    u32x4 v = {0u, 0u, 0u, 0u};
    if (head0 + hl < a.H && (p < 0 ? c < a.R : p < a.P))
      v = *(const u32x4*)((const uint16_t*)a.q + ((int64_t)row * a.H + head0 + hl) * RW + (p < 0 ? c : a.R + p));
    *(u32x4*)(qlds + hl * Lds::kQStride + c) = v;
  }
  const int seq = a.seq ? min(max(a.seq[row], 0), a.B - 1) : row;
  const int n = min(a.ctx[row], a.NB * a.BS);
  const int lo = a.window > 0 ? max(0, n - a.window) : 0;
  const int p0 = lo >> a.bs_shift;
  constexpr int KS = 4 * NCB;

  // every entry gets a valid page, whatever the context length says: no address rests on it
  for (int j = tid; j < a.lds_pages; j += 256) {
    const int p = p0 + j < a.NB ? a.table[(int64_t)seq * a.NB + p0 + j] : 0;
    pg[j] = (p >= 0 && p < a.num_pages) ? p : 0;
  }
  __syncthreads();
  // R may end inside the last column block: columns past it hold the row's start again, and meet
  // zeros in q or results that are not written
  int col_off[NCB];
#pragma unroll
  for (int cb = 0; cb < NCB; ++cb) {
    const int c = cb * 128 + l16 * 8;
    col_off[cb] = (c < a.R ? c : 0) * 2;
  }
  f32x4 o[HT][NCB * 8];
  float m[HT], l[HT];
#pragma unroll
  for (int ht = 0; ht < HT; ++ht) {
    m[ht] = -INFINITY;
    l[ht] = 0.f;
#pragma unroll
    for (int i = 0; i < NCB * 8; ++i) o[ht][i] = f32x4{0.f, 0.f, 0.f, 0.f};
  }
  const float sc = a.scale * 1.44269504088896f;
  const uint16_t* const qrow = qlds + (hwi * HT * 16 + l16) * Lds::kQStride + g * 8;
  const int mask = a.BS - 1;
  u32x4 v[NCB][8], kr[2][PK ? PK : 1];
  int rot_off[PK ? PK : 1];                   // past P: the part's start again, against zeros in q
#pragma unroll
  for (int ks = 0; ks < PK; ++ks) rot_off[ks] = (a.R + (ks * 32 + g * 8 < a.P ? ks * 32 + g * 8 : 0)) * 2;

  // Page of the visible keys of block b's half (16 keys lie in one page) and the range its rows are
  // clamped to: keys outside the visible range repeat a visible row, with weight zero.
  const char* base[2];
  int from[2], upto[2];
  auto locate = [&](int b) {
#pragma unroll
    for (int hf = 0; hf < 2; ++hf) {
      const int h0 = b * 32 + hf * 16;
      from[hf] = min(max(h0, lo), n - 1);
      upto[hf] = max(min(h0 + 15, n - 1), from[hf]);
      if (h0 + 15 < lo) upto[hf] = from[hf] = lo;
      const int page = __builtin_amdgcn_readfirstlane(pg[(from[hf] >> a.bs_shift) - p0]);
      base[hf] = (const char*)a.cache + (int64_t)page * a.BS * RW * 2;
    }
  };
  auto row_off = [&](int b, int i) {                             // bytes into the page
    const int hf = i >> 2;
    const int key = min(max(b * 32 + step_key(g, i), from[hf]), upto[hf]);
    return (uint32_t)((key & mask) * RW * 2);
  };
  auto load_rotated = [&](int b) {
#pragma unroll
    for (int hf = 0; hf < 2; ++hf) {
      const int key = min(max(b * 32 + hf * 16 + l16, from[hf]), upto[hf]);
      const uint32_t ro = (uint32_t)((key & mask) * RW * 2);
#pragma unroll
      for (int ks = 0; ks < PK; ++ks) kr[hf][ks] = *(const u32x4*)(base[hf] + (ro + rot_off[ks]));
    }
  };

  const int b1 = n > 0 ? (n - 1) >> 5 : -1, step = a.splits * kw;
  int b = (lo >> 5) + split * kw + kwi;
  if (b <= b1) {
    locate(b);
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      const uint32_t ro = row_off(b, i);
#pragma unroll
      for (int cb = 0; cb < NCB; ++cb) v[cb][i] = *(const u32x4*)(base[i >> 2] + (ro + col_off[cb]));
    }
    load_rotated(b);
  }
  for (; b <= b1; b += step) {
    const int k0 = b * 32;
    f32x4 s[HT][2];
#pragma unroll
    for (int hf = 0; hf < 2; ++hf) {
#pragma unroll
      for (int cb = 0; cb < NCB; ++cb)
#pragma unroll
        for (int i = 0; i < 4; ++i)
          *(u32x4*)(stage + (4 * g + i) * Lds::kStride + cb * 128 + l16 * 8) = v[cb][hf * 4 + i];
      __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
      __builtin_amdgcn_wave_barrier();
      __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
      f32x4 part[HT][2];                      // even and odd steps: two chains per head tile
#pragma unroll
      for (int ht = 0; ht < HT; ++ht) part[ht][0] = part[ht][1] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int ks = 0; ks < KS; ++ks) {
        const u32x4 kf = *(const u32x4*)(stage + l16 * Lds::kStride + ks * 32 + g * 8);
#pragma unroll
        for (int ht = 0; ht < HT; ++ht)
          part[ht][ks & 1] = mfma_bf16(kf, *(const u32x4*)(qrow + ht * 16 * Lds::kQStride + ks * 32), part[ht][ks & 1]);
      }
#pragma unroll
      for (int ks = 0; ks < PK; ++ks)
#pragma unroll
        for (int ht = 0; ht < HT; ++ht)
          part[ht][ks & 1] = mfma_bf16(kr[hf][ks], *(const u32x4*)(qrow + ht * 16 * Lds::kQStride + NCB * 128 + ks * 32),
                                       part[ht][ks & 1]);
#pragma unroll
      for (int ht = 0; ht < HT; ++ht) s[ht][hf] = part[ht][0] + part[ht][1];
      __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
      __builtin_amdgcn_wave_barrier();        // the stage is written again after these reads
      __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
    }
    u32x4 pf[HT];
#pragma unroll
    for (int ht = 0; ht < HT; ++ht) {
      float p[8], mx = -INFINITY;
#pragma unroll
      for (int i = 0; i < 8; ++i) p[i] = s[ht][i >> 2][i & 3] * sc;
      if (k0 < lo || k0 + 31 >= n) {
#pragma unroll
        for (int i = 0; i < 8; ++i) {
          const int key = k0 + step_key(g, i);
          if (key < lo || key >= n) p[i] = -INFINITY;
        }
      }
#pragma unroll
      for (int i = 0; i < 8; ++i) mx = fmaxf(mx, p[i]);
      mx = fmaxf(mx, lane_xor16(mx));
      mx = fmaxf(mx, lane_xor32(mx));
      const float mn = fmaxf(m[ht], mx);      // finite: every block holds a visible key
      const float f = __builtin_amdgcn_exp2f(m[ht] - mn);
      float sum = 0.f;
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        p[i] = __builtin_amdgcn_exp2f(p[i] - mn);
        sum += p[i];
      }
      l[ht] = l[ht] * f + sum;
      m[ht] = mn;
      if (__any(f != 1.f)) {
#pragma unroll
        for (int i = 0; i < NCB * 8; ++i) o[ht][i] *= f;
      }
      pf[ht] = u32x4{pack_bf16(p[0], p[1]), pack_bf16(p[2], p[3]), pack_bf16(p[4], p[5]),
                     pack_bf16(p[6], p[7])};
    }
    const int next = min(b + step, b1);       // after the last block its own rows again, unused
    locate(next);
    uint32_t ro[8];
#pragma unroll
    for (int i = 0; i < 8; ++i) ro[i] = row_off(next, i);
    load_rotated(next);
#pragma unroll
    for (int cb = 0; cb < NCB; ++cb) {
#pragma unroll
      for (int t = 0; t < 8; ++t) {
        const u32x4 vf = column_of(v[cb], t);
#pragma unroll
        for (int ht = 0; ht < HT; ++ht) o[ht][cb * 8 + t] = mfma_bf16(vf, pf[ht], o[ht][cb * 8 + t]);
      }
#pragma unroll
      for (int i = 0; i < 8; ++i) v[cb][i] = *(const u32x4*)(base[i >> 2] + (ro[i] + col_off[cb]));
    }
  }

  // the waves meet in LDS, one head tile of each at a time: sums, maxima and partial results per
  // wave, then all threads combine those that split the keys of a head
  const int RS = a.R + 4, per = rows_merge_floats(a.R);
  float* const merge = (float*)shared;
#pragma unroll
  for (int ht = 0; ht < HT; ++ht) {
    l[ht] += lane_xor16(l[ht]);
    l[ht] += lane_xor32(l[ht]);
    __syncthreads();                              // what the LDS held before is used up
    {
      float* const dst = merge + wave * per;
      if (g == 0) { dst[16 * RS + l16] = m[ht]; dst[16 * RS + 16 + l16] = l[ht]; }
#pragma unroll
      for (int cb = 0; cb < NCB; ++cb)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int col = cb * 128 + (4 * g + i) * 8;
          if (col < a.R) {
            float* d = dst + l16 * RS + col;
            const f32x4* t = o[ht] + cb * 8;
            *(f32x4*)d = f32x4{t[0][i], t[1][i], t[2][i], t[3][i]};
            *(f32x4*)(d + 4) = f32x4{t[4][i], t[5][i], t[6][i], t[7][i]};
          }
        }
    }
    __syncthreads();
    // per head: the common maximum, each key part's factor (over its maximum's place) and the sum
    if (tid < hw * 16) {
      float* const src = merge + (tid >> 4) * per + 16 * RS + (tid & 15);   // wave k * hw + tile: key part k
      float mx = src[0];
      for (int k = 1; k < kw; ++k) mx = fmaxf(mx, src[k * hw * per]);
      const float ms = mx == -INFINITY ? 0.f : mx;
      float sum = 0.f;
      for (int k = 0; k < kw; ++k) {
        float* const at = src + k * hw * per;
        const float f = __builtin_amdgcn_exp2f(at[0] - ms);
        sum += at[16] * f;
        at[0] = f;
      }
      const float inv = a.splits > 1 ? 1.f : (sum > 0.f ? 1.f / sum : 0.f);
      for (int k = 0; k < kw; ++k) src[k * hw * per] *= inv;
      const int head = head0 + ((tid >> 4) * HT + ht) * 16 + (tid & 15);
      if (a.splits > 1 && head < a.H) {
        float* ml = a.part + (int64_t)a.n * a.H * a.splits * a.R + (((int64_t)row * a.H + head) * a.splits + split) * 2;
        ml[0] = mx;
        ml[1] = sum;
      }
    }
    __syncthreads();
#pragma unroll 1
    for (int it = tid; it < hw * 256 * NCB; it += 256) {
      const int hl = it / (16 * NCB), c = it % (16 * NCB) * 8;
      const int head = head0 + ((hl >> 4) * HT + ht) * 16 + (hl & 15);
      if (head >= a.H || c >= a.R) continue;
      const float* src = merge + (hl >> 4) * per;
      float r[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
      for (int k = 0; k < kw; ++k) {
        const float* part = src + k * hw * per;
        const float f = part[16 * RS + (hl & 15)];
        float x[8];
        Vec8<F32>::ld(part, (hl & 15) * RS + c, x);
#pragma unroll
        for (int i = 0; i < 8; ++i) r[i] += x[i] * f;
      }
      const int64_t item = (int64_t)row * a.H + head;
      if (a.splits == 1) Vec8<BF16>::st(a.out, item * a.R + c, r);
      else Vec8<F32>::st(a.part, (item * a.splits + split) * a.R + c, r);
    }
  }
}

__global__ __launch_bounds__(64) void latent_rows_combine_kernel(RowsArgs a) {
  const int64_t item = blockIdx.x;       // (row, head)
  const float* ml = a.part + (int64_t)a.n * a.H * a.splits * a.R + item * a.splits * 2;
  float mx = -INFINITY;
  for (int s = 0; s < a.splits; ++s) mx = fmaxf(mx, ml[2 * s]);
  if (mx == -INFINITY) mx = 0.f;
  float l = 0.f;
  for (int s = 0; s < a.splits; ++s) l += ml[2 * s + 1] * __builtin_amdgcn_exp2f(ml[2 * s] - mx);
  const float inv = l > 0.f ? 1.f / l : 0.f;
  for (int c = threadIdx.x * 8; c < a.R; c += 512) {
    float acc[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
    for (int s = 0; s < a.splits; ++s) {
      const float f = __builtin_amdgcn_exp2f(ml[2 * s] - mx) * inv;
      float v[8];
      Vec8<F32>::ld(a.part, (item * a.splits + s) * a.R + c, v);
#pragma unroll
      for (int i = 0; i < 8; ++i) acc[i] += v[i] * f;
    }
    Vec8<BF16>::st(a.out, item * a.R + c, acc);
  }
}

// One workgroup per (token, head), plain fp32 arithmetic, any R and P.
template <typename T>
__global__ __launch_bounds__(256) void latent_plain_kernel(RowsArgs a) {
  extern __shared__ __align__(16) char lds_raw[];
  float* q = (float*)lds_raw;              // R + P
  __shared__ float sc[256];
  __shared__ float red[4];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int row = blockIdx.x / a.H;
  const int RW = a.R + a.P;
  const int64_t qat = (int64_t)blockIdx.x * RW, oat = (int64_t)blockIdx.x * a.R;
  const int seq = a.seq ? min(max(a.seq[row], 0), a.B - 1) : row;
  const int n = min(a.ctx[row], a.NB * a.BS);
  const int lo = a.window > 0 ? max(0, n - a.window) : 0;
  for (int c = tid; c < RW; c += 256) q[c] = Elem<T>::ld(a.q, qat + c);
  auto key_at = [&](int t) -> int64_t {
    const int p = page_of(a, t);
    int page = a.table[(int64_t)seq * a.NB + p];
    if (page < 0 || page >= a.num_pages) page = 0;
    return ((int64_t)page * a.BS + (t - p * a.BS)) * RW;
  };
  constexpr int kCols = 16;                // columns per thread: R <= 4096
  float o[kCols];
#pragma unroll
  for (int i = 0; i < kCols; ++i) o[i] = 0.f;
  float m = -INFINITY, l = 0.f;
  for (int c0 = lo; c0 < n; c0 += 256) {
    const int cnt = min(256, n - c0);
    __syncthreads();                       // q is there; the last chunk's scores are used up
    for (int j = wave; j < cnt; j += 4) {
      const int64_t at = key_at(c0 + j);
      float acc = 0.f;
      for (int c = lane; c < RW; c += 64) acc = fmaf(q[c], Elem<T>::ld(a.cache, at + c), acc);
      acc = wave_sum(acc);
      if (lane == 0) sc[j] = acc * a.scale;
    }
    __syncthreads();
    float mx = tid < cnt ? sc[tid] : -INFINITY;
    mx = wave_max(mx);
    if (lane == 0) red[wave] = mx;
    __syncthreads();
    mx = fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3]));
    const float mn = fmaxf(m, mx);
    const float f = expf(m - mn);
    __syncthreads();
    const float p = tid < cnt ? expf(sc[tid] - mn) : 0.f;
    sc[tid] = p;
    const float s = wave_sum(p);
    if (lane == 0) red[wave] = s;
    __syncthreads();
    l = l * f + red[0] + red[1] + red[2] + red[3];
    m = mn;
#pragma unroll
    for (int i = 0; i < kCols; ++i) o[i] *= f;
    for (int j = 0; j < cnt; ++j) {
      const int64_t at = key_at(c0 + j);
      const float pj = sc[j];
#pragma unroll
      for (int i = 0; i < kCols; ++i) {
        const int c = tid + i * 256;
        if (c < a.R) o[i] = fmaf(pj, Elem<T>::ld(a.cache, at + c), o[i]);
      }
    }
  }
  const float inv = l > 0.f ? 1.f / l : 0.f;
#pragma unroll
  for (int i = 0; i < kCols; ++i) {
    const int c = tid + i * 256;
    if (c < a.R) Elem<T>::st(a.out, oat + c, o[i] * inv);
  }
}

constexpr int kMaxLdsPages = 4096, kMaxRotated = 64;

// Head tiles per wave, and waves of a workgroup on different heads.
int rows_ht(int H, int R) { return H > 16 && R <= 256 ? 2 : 1; }   // registers hold 2 x 256 columns
int rows_hw(int H, int R) {
  const int tiles = (H + 16 * rows_ht(H, R) - 1) / (16 * rows_ht(H, R));
  return tiles >= 4 ? 4 : (tiles >= 2 ? 2 : 1);
}

// Key ranges per token: enough workgroups to cover the chip, at least two 32-key steps per wave.
int rows_splits(int n, int H, int R, int window, int NB, int BS) {
  const int hw = rows_hw(H, R), kw = 4 / hw, per = 16 * rows_ht(H, R) * hw;
  const int groups = n * ((H + per - 1) / per);
  int64_t keys = (int64_t)NB * BS;
  if (window > 0 && window < keys) keys = window;
  const int steps = (int)((keys + 31) / 32);
  const int resident = (R + 127) / 128 * rows_ht(H, R) <= 2 ? 2 : 1;       // workgroups per CU
  int s = 256 * resident / (groups > 0 ? groups : 1);
  s = s < steps / (2 * kw) ? s : steps / (2 * kw);
  s = s < 32 ? s : 32;
  return s < 1 ? 1 : s;
}

template <int NCB, int HT, int PK> int launch_latent_rows(RowsArgs a, hipStream_t st) {
  const size_t merge = 4 * sizeof(float) * (size_t)rows_merge_floats(a.R);
  const size_t work = 4 * RowsLds<NCB, PK>::kStage + (size_t)a.hw * HT * RowsLds<NCB, PK>::kQ;
  const size_t smem = (((size_t)a.lds_pages * 4 + 15) & ~(size_t)15) + (merge > work ? merge : work);
  if (smem > 64 * 1024 &&
      hipFuncSetAttribute((const void*)latent_rows_kernel<NCB, HT, PK>, hipFuncAttributeMaxDynamicSharedMemorySize,
                          (int)smem) != hipSuccess) {
    zp_set_error("latent_rows_attention: cannot reserve %zu bytes of LDS", smem);
    return ZP_EHIP;
  }
  const int hgroups = (a.H + 16 * HT * a.hw - 1) / (16 * HT * a.hw);
  hipLaunchKernelGGL((latent_rows_kernel<NCB, HT, PK>), dim3((unsigned)a.n * hgroups * a.splits), dim3(256), smem, st, a);
  ZP_LAUNCH_CHECK();
  if (a.splits > 1) {
    hipLaunchKernelGGL(latent_rows_combine_kernel, dim3((unsigned)a.n * a.H), dim3(64), 0, st, a);
    ZP_LAUNCH_CHECK();
  }
  return ZP_OK;
}

}  // namespace


extern "C" int zp_latent_norm_store(const void* in, const float* q_weight, const float* c_weight,
                                    void* q_out, void* c_out, void* cache, const int32_t* slots,
                                    const int32_t* positions, const float* freqs, int32_t n, int32_t q_width,
                                    int32_t c_width, int32_t p_width, int32_t q_norm, int32_t c_norm,
                                    int32_t rot, int64_t num_slots, float eps, int32_t dtype, void* stream) {
  ZP_REQUIRE(n >= 0 && q_width > 0 && c_width >= 0 && q_norm > 0 && q_norm <= q_width && c_norm <= c_width &&
                 (c_width ? c_norm > 0 && num_slots > 0 : p_width == 0) && p_width >= 0 && rot >= 0 && rot % 2 == 0 &&
                 rot <= p_width, "latent_norm_store: bad dims");
  ZP_MODEL_DTYPE("latent_norm_store");
  if (q_width % 8 || c_width % 8 || p_width % 8 || q_width > 512 * kNormPieces || c_width > 512 * kNormPieces) {
    zp_set_error("latent_norm_store: ranks %d, %d, rotated part %d unsupported (multiples of 8, <= %d)", q_width, c_width,
                 p_width, 512 * kNormPieces);
    return ZP_EUNSUPPORTED;
  }
  if (n == 0) return ZP_OK;
  ZP_REQUIRE(in && q_weight && q_out && (!c_width || (c_weight && cache && slots)) && (!rot || (positions && freqs)),
             "latent_norm_store: null pointer");
  ZP_REQUIRE(aligned16(in) && aligned16(q_weight) && aligned16(c_weight) && aligned16(q_out) &&
                 aligned16(c_out) && aligned16(cache), "latent_norm_store: tensors must be 16-byte aligned");
  NormStoreArgs a = {in, q_weight, c_weight, q_out, c_out, cache, slots, positions, freqs, n, q_width, c_width, p_width,
                     q_norm, c_norm, rot / 2, num_slots, eps};
  const unsigned grid = (unsigned)(((c_width ? 2 : 1) * (int64_t)n + 3) / 4);
  hipStream_t st = (hipStream_t)stream;
  if (dtype == ZP_BF16) hipLaunchKernelGGL((latent_norm_store_kernel<BF16>), dim3(grid), dim3(256), 0, st, a);
  else hipLaunchKernelGGL((latent_norm_store_kernel<F32>), dim3(grid), dim3(256), 0, st, a);
  ZP_LAUNCH_CHECK();
  return ZP_OK;
}

extern "C" int zp_rotate_heads(void* x, const int32_t* positions, const float* freqs, int32_t n, int32_t H, int32_t head,
                               int32_t at, int32_t rot, int64_t x_stride, int32_t dtype, void* stream) {
  ZP_REQUIRE(n >= 0 && H > 0 && head > 0 && at >= 0 && rot >= 0 && rot % 2 == 0 && at + rot <= head &&
                 x_stride >= (int64_t)H * head, "rotate_heads: bad dims");
  ZP_MODEL_DTYPE("rotate_heads");
  if (rot > 2048) {
    zp_set_error("rotate_heads: %d rotated dimensions (<= 2048)", rot);
    return ZP_EUNSUPPORTED;
  }
  if (n == 0 || rot == 0) return ZP_OK;
  ZP_REQUIRE(x && positions && freqs, "rotate_heads: null pointer");
  RotateArgs a = {x, positions, freqs, n, H, head, at, rot / 2, x_stride};
  const unsigned grid = (unsigned)((n + kRotTokens - 1) / kRotTokens);
  const size_t smem = sizeof(float2) * kRotTokens * (rot / 2);
  hipStream_t st = (hipStream_t)stream;
  const bool wide = rot % 16 == 0 && head % 8 == 0 && at % 8 == 0 && x_stride % 8 == 0 && aligned16(x);
#define ZP_ROTATE(T)                                                                                          \
  do {                                                                                                        \
    if (wide) hipLaunchKernelGGL((rotate_heads_kernel<T, 8>), dim3(grid), dim3(256), smem, st, a);            \
    else hipLaunchKernelGGL((rotate_heads_kernel<T, 1>), dim3(grid), dim3(256), smem, st, a);                 \
  } while (0)
  if (dtype == ZP_BF16) ZP_ROTATE(BF16); else ZP_ROTATE(F32);
#undef ZP_ROTATE
  ZP_LAUNCH_CHECK();
  return ZP_OK;
}

extern "C" int zp_headwise_linear(const void* in, const void* w, void* out, const int32_t* positions,
                                  const float* freqs, int32_t n, int32_t H, int32_t K, int32_t M, int32_t tail,
                                  int32_t rot, int32_t dtype, void* stream) {
  ZP_REQUIRE(n >= 0 && H > 0 && K > 0 && M > 0 && tail >= 0 && rot >= 0 && rot % 2 == 0 && rot <= tail &&
                 (rot == 0 || (positions && freqs)), "headwise_linear: bad dims");
  ZP_MODEL_DTYPE("headwise_linear");
  if (K % 32 != 0 || M % 16 != 0 || tail % 8 != 0 || H > 65535) {
    zp_set_error("headwise_linear: K %d, M %d, tail %d unsupported (multiples of 32, 16, 8)", K, M, tail);
    return ZP_EUNSUPPORTED;
  }
  if (n == 0) return ZP_OK;
  ZP_REQUIRE(in && w && out && aligned16(in) && aligned16(w) && aligned16(out),
             "headwise_linear: null or unaligned pointer");
  HeadArgs a = {in, w, out, positions, freqs, n, H, K, M, tail, rot / 2};
  // as many tokens per wave (W is read once for them) as still leave two workgroups per CU
  const int64_t columns = (int64_t)((M + 63) / 64) * H;
  int tt = 4;
  while (tt > 1 && columns * ((n + 16 * tt - 1) / (16 * tt)) < 512) tt >>= 1;
  const dim3 grid((M + 63) / 64, H, (n + 16 * tt - 1) / (16 * tt));
  ZP_REQUIRE(grid.z <= 65535, "headwise_linear: too many tokens");
  hipStream_t st = (hipStream_t)stream;
#define ZP_HEADWISE(T)                                                                            \
  do {                                                                                            \
    if (tt == 4) hipLaunchKernelGGL((headwise_kernel<T, 4>), grid, dim3(256), 0, st, a);          \
    else if (tt == 2) hipLaunchKernelGGL((headwise_kernel<T, 2>), grid, dim3(256), 0, st, a);     \
    else hipLaunchKernelGGL((headwise_kernel<T, 1>), grid, dim3(256), 0, st, a);                  \
  } while (0)
  if (dtype == ZP_BF16) ZP_HEADWISE(BF16);
  else ZP_HEADWISE(F32);
#undef ZP_HEADWISE
  ZP_LAUNCH_CHECK();
  return ZP_OK;
}

extern "C" int64_t zp_latent_rows_workspace(int32_t n, int32_t H, int32_t R, int32_t window,
                                            int32_t NB, int32_t BS, int32_t dtype) {
  if (n < 0 || H <= 0 || R <= 0 || NB <= 0 || BS <= 0) return -1;
  if (dtype != ZP_BF16 || R > 512) return 0;
  const int s = rows_splits(n, H, R, window, NB, BS);
  return s == 1 ? 0 : (int64_t)n * H * s * (R + 2) * 4;
}

extern "C" int zp_latent_rows_attention(const void* q, const void* cache, const int32_t* table,
                                        const int32_t* context_lens, const int32_t* table_rows,
                                        void* out, int32_t n, int32_t H, int32_t R, int32_t P, int32_t BS,
                                        int32_t B, int32_t NB, int32_t num_pages, int32_t window,
                                        float scale, int32_t dtype, void* workspace,
                                        int64_t workspace_bytes, void* stream) {
  ZP_REQUIRE(n >= 0 && H > 0 && R > 0 && P >= 0 && BS > 0 && B > 0 && NB > 0 && num_pages > 0 && window >= 0,
             "latent_rows_attention: bad dims");
  ZP_MODEL_DTYPE("latent_rows_attention");
  if (R % 32 != 0 || R > 4096 || P % 8 != 0 || P > 4096) {
    zp_set_error("latent_rows_attention: latent size %d, rotated part %d unsupported (multiples of 32 and 8, <= 4096)", R, P);
    return ZP_EUNSUPPORTED;
  }
  if (n == 0) return ZP_OK;
  ZP_REQUIRE(q && cache && table && context_lens && out, "latent_rows_attention: null pointer");
  ZP_REQUIRE(table_rows || n <= B, "latent_rows_attention: more tokens than table rows");
  ZP_REQUIRE(aligned16(q) && aligned16(cache) && aligned16(out) && aligned16(workspace),
             "latent_rows_attention: tensors must be 16-byte aligned");
  RowsArgs a = {};
  a.q = q; a.cache = cache; a.table = table; a.ctx = context_lens; a.seq = table_rows; a.out = out;
  a.part = (float*)workspace; a.n = n; a.H = H; a.R = R; a.P = P; a.BS = BS; a.B = B; a.NB = NB;
  a.num_pages = num_pages; a.window = window; a.scale = scale; a.bs_shift = -1;
  if ((BS & (BS - 1)) == 0)
    for (a.bs_shift = 0; (1 << a.bs_shift) < BS; ++a.bs_shift) {}
  int64_t pages = NB;
  if (window > 0 && (window - 1) / BS + 2 < pages) pages = (window - 1) / BS + 2;
  hipStream_t st = (hipStream_t)stream;
  if (dtype == ZP_F32 || R > 512 || P > kMaxRotated || pages > kMaxLdsPages || a.bs_shift < 4) {   // bs_shift -1: not a power of two
    const size_t smem = sizeof(float) * (R + P);
    if (dtype == ZP_BF16)
      hipLaunchKernelGGL((latent_plain_kernel<BF16>), dim3((unsigned)n * H), dim3(256), smem, st, a);
    else
      hipLaunchKernelGGL((latent_plain_kernel<F32>), dim3((unsigned)n * H), dim3(256), smem, st, a);
    ZP_LAUNCH_CHECK();
    return ZP_OK;
  }
  a.hw = rows_hw(H, R);
  a.lds_pages = (int)pages;
  a.splits = rows_splits(n, H, R, window, NB, BS);
  ZP_REQUIRE(a.splits == 1 || (workspace && workspace_bytes >= zp_latent_rows_workspace(n, H, R, window, NB, BS, dtype)),
             "latent_rows_attention: workspace too small");
  const bool two = rows_ht(H, R) == 2;
#define ZP_LATENT_ROWS(NCB, HT) (P ? launch_latent_rows<NCB, HT, 2>(a, st) : launch_latent_rows<NCB, HT, 0>(a, st))
  switch ((R + 127) / 128) {
    case 1: return two ? ZP_LATENT_ROWS(1, 2) : ZP_LATENT_ROWS(1, 1);
    case 2: return two ? ZP_LATENT_ROWS(2, 2) : ZP_LATENT_ROWS(2, 1);
    case 3: return ZP_LATENT_ROWS(3, 1);
    default: return ZP_LATENT_ROWS(4, 1);
  }
#undef ZP_LATENT_ROWS
}
