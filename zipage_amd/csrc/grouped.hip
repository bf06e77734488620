// Grouped-query attention over paged rows [keys of all heads | values of all heads] per token.
//
//   rotary_store    rotary positions on queries and keys, and on values where those turn too; norms over
//                   the whole projections before that; keys and values to their cache slot
//   grouped_rows    attention of single tokens over the pages; the query heads of a key head share
//                   one read of its keys and values
//   grouped_plain   float32 form (true fp32 products), any sizes
//
// Attention of runs of prompt tokens is run_attention (runs.hip).  A token sees a window, its own
// block of positions, or everything before it; a sink is a logit per head that joins the softmax's
// denominator only.  A head may hold two maps over the same values (differential attention): in
// grouped_rows they are two query columns of a key head of twice the length, each with zeros where the
// other one's elements are, so that keys and values are still read once.  Values that turned with their
// position turn back with the query's in the last step of a kernel.
#include "mfma.h"

namespace {

// ------------------------------------------------------------------ rotary positions and the store
struct RotaryArgs {
  const void* in;           // token rows of in_st elements: q (H * D), k (HK * D), v (VT)
  const float* bias;        // the same row, added before the turn; or null
  const int32_t* positions;
  const float* freqs;       // (rot / 2,)
  void* q_out;              // (n, H * D)
  void* kv_out;             // (n, HK * D + VT) or null
  void* cache;              // (num_slots, HK * D + VT)
  const int32_t* slots;     // (n,), -1 skips
  int n, H, HK, D, VT, half; // half = rotated dimensions / 2
  int64_t in_st, num_slots;
  // what only some designs have
  const float* norm;        // (H * D + HK * D,) weights of RMS norms over all of q and all of k, or null
  int q_norm, k_norm;       // lengths of their means
  float eps;
  bool tied;                // the values are the keys as projected; rows of `in` end with k
  int V;                    // of a value head
  const float* vfreqs;      // (V / 2,): values turn, elements 2 i and 2 i + 1 with frequency i; or null
  float2* turns;            // (n, V / 2): cos and sin of the values' angles, for the way back
  int staged;               // bytes of q and k that wait in LDS while their norms are taken; 0: they are read twice
};

// Four tokens per workgroup, or one where there are few, each with its own threads; a token's angles once, in LDS, for
// all heads.  VEC elements per item; an item of the rotated part is the pair (i .. i + VEC, i + half ..).  NORM: norms
// over q and k, and tied values; TURN: values turn.
template <typename T, int VEC, int TOKENS, bool NORM, bool TURN>
__global__ __launch_bounds__(256) void rotary_store_kernel(RotaryArgs a) {
  extern __shared__ __align__(16) char lds_raw[];
  __shared__ float squares[2][4];           // of q and k, by wave
  constexpr int kPer = 256 / TOKENS;        // threads per token
  const int tok = TOKENS == 1 ? 0 : __builtin_amdgcn_readfirstlane(threadIdx.x / kPer), tid = threadIdx.x % kPer;
  const int64_t row = blockIdx.x * TOKENS + tok;
  const bool live = row < a.n;              // uniform in the wave
  const int heads = a.H + a.HK, edge = a.H * a.D, end = heads * a.D;
  float2* const cs = (float2*)lds_raw + tok * a.half;                        // [TOKENS][half]
  float2* const vcs = (float2*)lds_raw + TOKENS * a.half + tok * (a.V / 2);   // [TOKENS][V / 2]
  char* const wait = lds_raw + ((TOKENS * (a.half + (TURN ? a.V / 2 : 0)) * 8 + 15) & ~15) + tok * a.staged;   // [TOKENS][staged]
  if (live) {
    typename Vec8<T>::Raw x[4];              // pieces of q and k, requested while the angles are computed
    auto fetch = [&](int c0) {
#pragma unroll
      for (int u = 0; u < 4; ++u) x[u] = Vec8<T>::raw(a.in, row * a.in_st + min(c0 + u * kPer * 8, end - 8));
    };
    if (NORM && a.norm) fetch(tid * 8);
    const int position = a.positions[row];
    for (int i = tid; i < a.half; i += kPer) cs[i] = rotary_turn(position, a.freqs[i]);
    if (TURN)
      for (int i = tid; i < a.V / 2; i += kPer) {
        vcs[i] = rotary_turn(position, a.vfreqs[i]);
        a.turns[row * (a.V / 2) + i] = vcs[i];
      }
    if (NORM && a.norm) {
      float qs = 0.f, ks = 0.f;
      for (int c0 = tid * 8; c0 < end; c0 += 4 * kPer * 8) {
#pragma unroll
        for (int u = 0; u < 4; ++u) {
          const int c = c0 + u * kPer * 8;
          float v[8], s = 0.f;
          Vec8<T>::unpack(x[u], v);
#pragma unroll
          for (int i = 0; i < 8; ++i) s = fmaf(v[i], v[i], s);
          if (c < edge) qs += s; else if (c < end) ks += s;
          if (a.staged && c < end) Vec8<T>::st(wait, c, v);
        }
        if (c0 + 4 * kPer * 8 < end) fetch(c0 + 4 * kPer * 8);
      }
      qs = wave_sum(qs);
      ks = wave_sum(ks);
      if ((threadIdx.x & 63) == 0) {
        squares[0][threadIdx.x >> 6] = qs;
        squares[1][threadIdx.x >> 6] = ks;
      }
    }
  }
  __syncthreads();
  if (!live) return;
  float rq = 1.f, rk = 1.f;
  if (NORM && a.norm) {
    float qs = 0.f, ks = 0.f;
#pragma unroll
    for (int w = 0; w < 4 / TOKENS; ++w) {
      qs += squares[0][tok * (4 / TOKENS) + w];
      ks += squares[1][tok * (4 / TOKENS) + w];
    }
    rq = 1.f / sqrtf(qs / (float)a.q_norm + a.eps);
    rk = 1.f / sqrtf(ks / (float)a.k_norm + a.eps);
  }
  const int pairs = a.half / VEC, per_head = (a.D - a.half) / VEC;
  const int rotated = heads * per_head, items = rotated + a.VT / VEC;
  const uint32_t inv = 0xffffffffu / per_head + 1;           // of a division; per_head 1 overflows to 0
  const int kvw = a.HK * a.D + a.VT;
  int64_t slot = a.slots[row];
  if (slot >= a.num_slots) slot = -1;
  auto raw = [&](int c, float* o) {
    if (NORM && a.staged && c < end) {
      if constexpr (VEC == 8) Vec8<T>::ld(wait, c, o); else o[0] = Elem<T>::ld(wait, c);
      return;
    }
    const int64_t at = row * a.in_st + c;
    if constexpr (VEC == 8) Vec8<T>::ld(a.in, at, o); else o[0] = Elem<T>::ld(a.in, at);
    if (!NORM && a.bias) {
      float b[VEC];
      if constexpr (VEC == 8) Vec8<F32>::ld(a.bias, c, b); else b[0] = a.bias[c];
#pragma unroll
      for (int i = 0; i < VEC; ++i) o[i] += b[i];
    }
  };
  auto load = [&](int c, float* o) {         // of q or k
    raw(c, o);
    if (NORM && a.norm) {
      float w[VEC];
      if constexpr (VEC == 8) Vec8<F32>::ld(a.norm, c, w); else w[0] = a.norm[c];
      const float r = c < edge ? rq : rk;
#pragma unroll
      for (int i = 0; i < VEC; ++i) o[i] *= r * w[i];
    }
  };
  auto put = [&](int c, const float* o) {   // column of the row [q | k | v]
    const int kc = c - edge;
    if (kc < 0) {
      if constexpr (VEC == 8) Vec8<T>::st(a.q_out, row * edge + c, o);
      else Elem<T>::st(a.q_out, row * edge + c, o[0]);
      return;
    }
    if (a.kv_out) {
      if constexpr (VEC == 8) Vec8<T>::st(a.kv_out, row * kvw + kc, o);
      else Elem<T>::st(a.kv_out, row * kvw + kc, o[0]);
    }
    if (slot >= 0) {
      if constexpr (VEC == 8) Vec8<T>::st(a.cache, slot * kvw + kc, o);
      else Elem<T>::st(a.cache, slot * kvw + kc, o[0]);
    }
  };
  for (int it = tid; it < items; it += kPer) {
    float x[VEC], y[VEC];
    if (it >= rotated) {
      const int v = (it - rotated) * VEC, c = end + v;
      const int from = NORM && a.tied ? edge + v : c;
      raw(from, x);
      if (TURN) {
        const float2* r = vcs + v % a.V / 2;
        if constexpr (VEC == 8) {
#pragma unroll
          for (int i = 0; i < 4; ++i) turn_pair(x[2 * i], x[2 * i + 1], r[i].x, r[i].y);
        } else {
          raw(from ^ 1, y);                    // heads start at even columns
          x[0] = v & 1 ? x[0] * r->x + y[0] * r->y : x[0] * r->x - y[0] * r->y;
        }
      }
      put(c, x);
      continue;
    }
    const int h = per_head == 1 ? it : (int)__umulhi((uint32_t)it, inv), p = it - h * per_head;
    if (p >= pairs) {                          // dimensions behind the rotated ones
      const int c = h * a.D + (p + pairs) * VEC;
      load(c, x);
      put(c, x);
      continue;
    }
    const int c = h * a.D + p * VEC;
    load(c, x);
    load(c + a.half, y);
#pragma unroll
    for (int i = 0; i < VEC; ++i) {
      const float2 r = cs[p * VEC + i];
      turn_pair(x[i], y[i], r.x, r.y);
    }
    put(c, x);
    put(c + a.half, y);
  }
}

// ------------------------------------------------------------------ single tokens over the pages
struct RowsArgs {
  const void* q;          // (n, H * D / maps)
  const void* cache;      // (pages, BS, HK * (D + V))
  const int32_t* table;   // (B, NB) page ids
  const int32_t* ctx;     // (n,) tokens of the sequence up to and including this one; 0 = inert
  const int32_t* seq;     // (n,) row of table, or null: row i
  const float* sinks;     // (H,) or null
  void* out;              // token rows of o_st elements, head h at h * V
  float* part;            // splits > 1: (n, H, splits, V) fp32, then (n, H, splits, 2) max and sum
  int n, H, HK, D, V, BS, bs_shift, B, NB, num_pages;   // H counts the maps of a head, D is a key head's length
  int window, chunk;
  int splits, htiles;     // key ranges, and tiles of 16 query heads per key head
  int lds_pages;
  int64_t o_st;
  float scale, out_scale;
  float cap;              // > 0: soft cap of the scores
  // two maps: rms(o1 - balance * o2) * out_scale * sigmoid(gate), the mean over vdim
  float balance, eps;
  int vdim;
  const void* gate;       // token rows of g_st elements, head h at h * V; or null
  int64_t g_st;
  const float2* turns;    // one map: (n, V / 2) cos and sin, results turn back by them; or null
};

// A piece of a head's result, normed: scale and gate it, and store it.
template <typename T> __device__ __forceinline__ void store_gated(const RowsArgs& a, int64_t row, int head, int c, float* r, float scale) {
#pragma unroll
  for (int i = 0; i < 8; ++i) r[i] *= scale;
  if (a.gate) {
    float z[8];
    Vec8<T>::ld(a.gate, row * a.g_st + (int64_t)head * a.V + c, z);
#pragma unroll
    for (int i = 0; i < 8; ++i) r[i] *= sigmoid_of<T>(z[i]);
  }
  Vec8<T>::st(a.out, row * a.o_st + (int64_t)head * a.V + c, r);
}

__device__ __forceinline__ int first_key(const RowsArgs& a, int n) {   // n tokens, the last one asks
  if (a.window > 0) return max(0, n - a.window);
  return a.chunk > 0 && n > 0 ? (n - 1) / a.chunk * a.chunk : 0;
}

// A workgroup owns one token, up to 16 query heads of one key head and one key range; its four waves
// are flash loops of their own over every fourth 32-key step and meet in LDS at the end.  Keys are the
// row operand straight from memory (64-byte pieces), values are loaded as rows and turned into column
// operands by v_perm.  The next step's keys are requested once the scores are done, its values once the
// value products are.
template <int DKS, int VCB, int MAPS>
__global__ __launch_bounds__(256, 2) void grouped_rows_kernel(RowsArgs a) {
  extern __shared__ __align__(16) char lds_raw[];
  int* const pg = (int*)lds_raw;
  float* const merge = (float*)(lds_raw + ((a.lds_pages * 4 + 15) & ~15));
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l16 = lane & 15, g = lane >> 4;
  int id = blockIdx.x;
  const int split = id % a.splits;
  id /= a.splits;
  const int ht = id % a.htiles;
  id /= a.htiles;
  const int hk = id % a.HK, row = id / a.HK;
  const int G = a.H / a.HK;
  const int seq = a.seq ? min(max(a.seq[row], 0), a.B - 1) : row;
  const int n = min(a.ctx[row], a.NB * a.BS);
  const int lo = first_key(a, n);
  const int p0 = lo >> a.bs_shift;
  // every entry gets a valid page, whatever the context length says: no address rests on it
  for (int j = tid; j < a.lds_pages; j += 256) {
    const int p = p0 + j < a.NB ? a.table[(int64_t)seq * a.NB + p0 + j] : 0;
    pg[j] = (p >= 0 && p < a.num_pages) ? p : 0;
  }
  const int head = hk * G + min(ht * 16 + l16, G - 1), qd = a.D / MAPS;
  u32x4 qf[DKS];
  const uint16_t* q = (const uint16_t*)a.q + ((int64_t)row * a.H + head) * qd;
#pragma unroll
  for (int ks = 0; ks < DKS; ++ks) {
    const int c = ks * 32 + g * 8 - (MAPS == 2 ? (head & 1) * qd : 0);     // element of this map
    const bool own = c >= 0 && c < qd;
    qf[ks] = *(const u32x4*)(q + (own ? c : 0));
    if (!own) qf[ks] = u32x4{0u, 0u, 0u, 0u};
  }
  // key columns past the head's end repeat its start, against zeros in q
  const int nks = a.D / 32, past = -g * 8, tail = nks * 32 + g * 8 < a.D ? nks * 32 : past;
  __syncthreads();
  const int kvw = a.HK * (a.D + a.V), mask = a.BS - 1;
  const uint16_t* const kc = (const uint16_t*)a.cache + hk * a.D + g * 8;
  const uint16_t* const vc = (const uint16_t*)a.cache + a.HK * a.D + hk * a.V;
  int col[VCB];
#pragma unroll
  for (int cb = 0; cb < VCB; ++cb) {
    const int c = cb * 128 + l16 * 8;
    col[cb] = c < a.V ? c : 0;
  }
  // keys outside the visible range repeat a visible row, with weight zero
  auto row_at = [&](int key) -> int64_t {
    key = min(max(key, lo), n - 1);
    const int page = pg[min((key >> a.bs_shift) - p0, a.lds_pages - 1)];
    return ((int64_t)page * a.BS + (key & mask)) * kvw;
  };
  u32x4 kf[2][DKS], vf[VCB][8];
  auto load_keys = [&](int b) {
#pragma unroll
    for (int tt = 0; tt < 2; ++tt) {
      const uint16_t* k = kc + row_at(b * 32 + tt * 16 + l16);
#pragma unroll
      for (int ks = 0; ks < DKS; ++ks) kf[tt][ks] = *(const u32x4*)(k + (ks < nks ? ks * 32 : (ks == nks ? tail : past)));
    }
  };
  auto load_values = [&](int b) {
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      const uint16_t* v = vc + row_at(b * 32 + step_key(g, i));
#pragma unroll
      for (int cb = 0; cb < VCB; ++cb) vf[cb][i] = *(const u32x4*)(v + col[cb]);
    }
  };
  f32x4 o[VCB * 8];
#pragma unroll
  for (int i = 0; i < VCB * 8; ++i) o[i] = f32x4{0.f, 0.f, 0.f, 0.f};
  const SoftCap cap(a.scale, a.cap);
  float m = cap.bounded ? 0.f : -INFINITY, l = 0.f;
  const int b1 = n > 0 ? (n - 1) >> 5 : -1, step = 4 * a.splits;
  int b = (lo >> 5) + split * 4 + wave;
  if (b <= b1) {
    load_keys(b);
    load_values(b);
  }
  for (; b <= b1; b += step) {
    const int k0 = b * 32, next = min(b + step, b1);       // after the last step its own rows again, unused
    f32x4 s[2];
#pragma unroll
    for (int tt = 0; tt < 2; ++tt) {
      s[tt] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int ks = 0; ks < DKS; ++ks) s[tt] = mfma_bf16(kf[tt][ks], qf[ks], s[tt]);
    }
    load_keys(next);
    float p[8], sum = 0.f;
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      const int key = k0 + step_key(g, i);
      p[i] = cap.log2_score(s[i >> 2][i & 3]);
      if (key < lo || key >= n) p[i] = -INFINITY;
    }
    if (!cap.bounded) {
      float mx = -INFINITY;
#pragma unroll
      for (int i = 0; i < 8; ++i) mx = fmaxf(mx, p[i]);
      mx = fmaxf(mx, lane_xor16(mx));
      mx = fmaxf(mx, lane_xor32(mx));
      const float mn = fmaxf(m, mx);                        // finite: every step holds a visible key
      const float f = __builtin_amdgcn_exp2f(m - mn);
#pragma unroll
      for (int i = 0; i < 8; ++i) p[i] -= mn;
      l *= f;
      m = mn;
      if (__any(f != 1.f)) {
#pragma unroll
        for (int i = 0; i < VCB * 8; ++i) o[i] *= f;
      }
    }
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      p[i] = __builtin_amdgcn_exp2f(p[i]);
      sum += p[i];
    }
    l += sum;
    const u32x4 pf = {pack_bf16(p[0], p[1]), pack_bf16(p[2], p[3]), pack_bf16(p[4], p[5]), pack_bf16(p[6], p[7])};
#pragma unroll
    for (int cb = 0; cb < VCB; ++cb)
#pragma unroll
      for (int t = 0; t < 8; ++t) o[cb * 8 + t] = mfma_bf16(column_of(vf[cb], t), pf, o[cb * 8 + t]);
    load_values(next);
  }
  l += lane_xor16(l);
  l += lane_xor32(l);
  const int RS = a.V + 4, per = 16 * RS + 32;
  float* const dst = merge + wave * per;
  if (g == 0) { dst[16 * RS + l16] = m; dst[16 * RS + 16 + l16] = l; }
#pragma unroll
  for (int cb = 0; cb < VCB; ++cb)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int c = cb * 128 + (4 * g + i) * 8;
      if (c < a.V) {
        float* d = dst + l16 * RS + c;
        const f32x4* t = o + cb * 8;
        *(f32x4*)d = f32x4{t[0][i], t[1][i], t[2][i], t[3][i]};
        *(f32x4*)(d + 4) = f32x4{t[4][i], t[5][i], t[6][i], t[7][i]};
      }
    }
  __syncthreads();
  if (tid < 16 && ht * 16 + tid < G) {
    const int h = hk * G + ht * 16 + tid;
    float* const src = merge + 16 * RS + tid;
    float mx = fmaxf(fmaxf(src[0], src[per]), fmaxf(src[2 * per], src[3 * per]));
    const float ms = mx == -INFINITY ? 0.f : mx;
    float sum = 0.f, f[4];
#pragma unroll
    for (int k = 0; k < 4; ++k) {
      f[k] = __builtin_amdgcn_exp2f(src[k * per] - ms);
      sum += src[k * per + 16] * f[k];
    }
    float inv = 1.f;
    if (a.splits > 1) {
      float* ml = a.part + (int64_t)a.n * a.H * a.splits * a.V + (((int64_t)row * a.H + h) * a.splits + split) * 2;
      ml[0] = mx;
      ml[1] = sum;
    } else {
      if (a.sinks && mx != -INFINITY) sum += __builtin_amdgcn_exp2f(a.sinks[h] * 1.44269504088896f - ms);
      inv = sum > 0.f ? (MAPS == 1 ? a.out_scale : 1.f) / sum : 0.f;
    }
#pragma unroll
    for (int k = 0; k < 4; ++k) src[k * per] = f[k] * inv;
  }
  __syncthreads();
  if (MAPS == 2 && a.splits == 1) {              // a wave per head, a lane per eight columns
    for (int pr = wave; pr < 8 && ht * 16 + 2 * pr < G; pr += 4) {
      const int c = lane * 8;
      float r[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f}, ss = 0.f;
      if (c < a.V) {
#pragma unroll
        for (int k = 0; k < 8; ++k) {            // four waves' parts of the two maps
          const float* part = merge + (k >> 1) * per;
          const int hl = 2 * pr + (k & 1);
          const float f = part[16 * RS + hl] * ((k & 1) ? -a.balance : 1.f);
          float x[8];
          Vec8<F32>::ld(part, hl * RS + c, x);
#pragma unroll
          for (int i = 0; i < 8; ++i) r[i] += x[i] * f;
        }
#pragma unroll
        for (int i = 0; i < 8; ++i) ss += r[i] * r[i];
      }
      ss = wave_sum(ss);
      if (c < a.V) store_gated<BF16>(a, row, (hk * G + ht * 16) / 2 + pr, c, r, a.out_scale / sqrtf(ss / (float)a.vdim + a.eps));
    }
    return;
  }
  for (int it = tid; it < 16 * (a.V / 8); it += 256) {
    const int hl = it / (a.V / 8), c = (it - hl * (a.V / 8)) * 8;
    if (ht * 16 + hl >= G) continue;
    const int h = hk * G + ht * 16 + hl;
    float r[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int k = 0; k < 4; ++k) {
      const float* part = merge + k * per;
      const float f = part[16 * RS + hl];
      float x[8];
      Vec8<F32>::ld(part, hl * RS + c, x);
#pragma unroll
      for (int i = 0; i < 8; ++i) r[i] += x[i] * f;
    }
    if (a.splits == 1) {
      if (a.turns) turn_back8(r, a.turns + ((int64_t)row * a.V + c) / 2);
      Vec8<BF16>::st(a.out, row * a.o_st + (int64_t)h * a.V + c, r);
    } else Vec8<F32>::st(a.part, (((int64_t)row * a.H + h) * a.splits + split) * a.V + c, r);
  }
}

__global__ __launch_bounds__(64) void grouped_combine_kernel(RowsArgs a) {
  const int64_t item = blockIdx.x;       // (row, head)
  const int h = (int)(item % a.H);
  const float* ml = a.part + (int64_t)a.n * a.H * a.splits * a.V + item * a.splits * 2;
  float mx = -INFINITY;
  for (int s = 0; s < a.splits; ++s) mx = fmaxf(mx, ml[2 * s]);
  const bool any = mx != -INFINITY;
  if (!any) mx = 0.f;
  float l = 0.f;
  for (int s = 0; s < a.splits; ++s) l += ml[2 * s + 1] * __builtin_amdgcn_exp2f(ml[2 * s] - mx);
  if (a.sinks && any) l += __builtin_amdgcn_exp2f(a.sinks[h] * 1.44269504088896f - mx);
  const float inv = l > 0.f ? a.out_scale / l : 0.f;
  for (int c = threadIdx.x * 8; c < a.V; c += 512) {
    float acc[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
    for (int s = 0; s < a.splits; ++s) {
      const float f = __builtin_amdgcn_exp2f(ml[2 * s] - mx) * inv;
      float v[8];
      Vec8<F32>::ld(a.part, (item * a.splits + s) * a.V + c, v);
#pragma unroll
      for (int i = 0; i < 8; ++i) acc[i] += v[i] * f;
    }
    if (a.turns) turn_back8(acc, a.turns + (item / a.H * a.V + c) / 2);
    Vec8<BF16>::st(a.out, item / a.H * a.o_st + (int64_t)h * a.V + c, acc);
  }
}

// The two maps of a head (V <= 512).
__global__ __launch_bounds__(64) void grouped_pair_combine_kernel(RowsArgs a) {
  const int heads = a.H / 2, row = blockIdx.x / heads, head = blockIdx.x - row * heads;
  const int c = threadIdx.x * 8;
  float r[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f}, ss = 0.f;
  for (int map = 0; map < 2; ++map) {
    const int64_t item = (int64_t)row * a.H + head * 2 + map;
    const float* ml = a.part + (int64_t)a.n * a.H * a.splits * a.V + item * a.splits * 2;
    float mx = -INFINITY, l = 0.f;
    for (int s = 0; s < a.splits; ++s) mx = fmaxf(mx, ml[2 * s]);
    if (mx == -INFINITY) mx = 0.f;
    for (int s = 0; s < a.splits; ++s) l += ml[2 * s + 1] * __builtin_amdgcn_exp2f(ml[2 * s] - mx);
    const float inv = l > 0.f ? (map ? -a.balance : 1.f) / l : 0.f;
    if (c < a.V)
      for (int s = 0; s < a.splits; ++s) {
        const float f = __builtin_amdgcn_exp2f(ml[2 * s] - mx) * inv;
        float v[8];
        Vec8<F32>::ld(a.part, (item * a.splits + s) * a.V + c, v);
#pragma unroll
        for (int i = 0; i < 8; ++i) r[i] += v[i] * f;
      }
  }
#pragma unroll
  for (int i = 0; i < 8; ++i) ss += r[i] * r[i];
  ss = wave_sum(ss);
  if (c < a.V) store_gated<BF16>(a, row, head, c, r, a.out_scale / sqrtf(ss / (float)a.vdim + a.eps));
}

// One workgroup per (token, head), plain fp32 arithmetic; two maps one after the other.
template <typename T, int MAPS>
__global__ __launch_bounds__(256) void grouped_plain_kernel(RowsArgs a) {
  extern __shared__ __align__(16) char lds_raw[];
  float* q = (float*)lds_raw;              // D
  __shared__ float sc[256];
  __shared__ float red[4];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int heads = a.H / MAPS, row = blockIdx.x / heads, h = blockIdx.x - row * heads, hk = h / (heads / a.HK);
  const int seq = a.seq ? min(max(a.seq[row], 0), a.B - 1) : row;
  const int n = min(a.ctx[row], a.NB * a.BS), qd = a.D / MAPS;
  const int lo = first_key(a, n);
  const int64_t kvw = (int64_t)a.HK * (a.D + a.V);
  auto key_at = [&](int t) -> int64_t {
    const int p = a.bs_shift >= 0 ? t >> a.bs_shift : t / a.BS;
    int page = a.table[(int64_t)seq * a.NB + p];
    if (page < 0 || page >= a.num_pages) page = 0;
    return ((int64_t)page * a.BS + (t - p * a.BS)) * kvw;
  };
  constexpr int kCols = 4;                 // columns per thread: V <= 1024
  float total[kCols] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll 1
  for (int map = 0; map < MAPS; ++map) {
    __syncthreads();                       // the map before is done with q and its scores
    for (int c = tid; c < qd; c += 256) q[c] = Elem<T>::ld(a.q, ((int64_t)blockIdx.x * MAPS + map) * qd + c);
    float o[kCols] = {0.f, 0.f, 0.f, 0.f};
    float m = -INFINITY, l = 0.f;
    for (int c0 = lo; c0 < n; c0 += 256) {
      const int cnt = min(256, n - c0);
      __syncthreads();                     // q is there; the last chunk's scores are used up
      for (int j = wave; j < cnt; j += 4) {
        const int64_t at = key_at(c0 + j) + hk * a.D + map * qd;
        float acc = 0.f;
        for (int c = lane; c < qd; c += 64) acc = fmaf(q[c], Elem<T>::ld(a.cache, at + c), acc);
        acc = wave_sum(acc) * a.scale;
        if (a.cap > 0.f) acc = a.cap * tanhf(acc / a.cap);
        if (lane == 0) sc[j] = acc;
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
        const int64_t at = key_at(c0 + j) + a.HK * a.D + hk * a.V;
        const float pj = sc[j];
#pragma unroll
        for (int i = 0; i < kCols; ++i) {
          const int c = tid + i * 256;
          if (c < a.V) o[i] = fmaf(pj, Elem<T>::ld(a.cache, at + c), o[i]);
        }
      }
    }
    if (MAPS == 1 && a.sinks && n > 0) l += expf(a.sinks[h] - m);
    const float inv = l > 0.f ? 1.f / l : 0.f;
#pragma unroll
    for (int i = 0; i < kCols; ++i) total[i] += o[i] * inv * (map ? -a.balance : 1.f);
  }
  float scale = a.out_scale;
  if constexpr (MAPS == 2) {
    float ss = 0.f;                        // columns past V are zero
#pragma unroll
    for (int i = 0; i < kCols; ++i) ss += total[i] * total[i];
    ss = wave_sum(ss);
    __syncthreads();
    if (lane == 0) red[wave] = ss;
    __syncthreads();
    scale /= sqrtf((red[0] + red[1] + red[2] + red[3]) / (float)a.vdim + a.eps);
  }
#pragma unroll
  for (int i = 0; i < kCols; ++i) {
    const int c = tid + i * 256;
    if (c >= a.V) continue;
    float r = total[i] * scale;
    if (MAPS == 1 && a.turns) {              // the pair's other element is the neighbouring lane's
      const float other = __shfl_xor(r, 1);
      const float2 t = a.turns[((int64_t)row * a.V + c) / 2];
      r = c & 1 ? r * t.x - other * t.y : r * t.x + other * t.y;
    }
    if (MAPS == 2 && a.gate) r *= sigmoid_of<T>(Elem<T>::ld(a.gate, row * a.g_st + (int64_t)h * a.V + c));
    Elem<T>::st(a.out, row * a.o_st + (int64_t)h * a.V + c, r);
  }
}

constexpr int kMaxLdsPages = 4096;

// Key ranges per token: enough workgroups to cover the chip, at least two steps per wave.
int rows_splits(int n, int H, int HK, int window, int chunk, int NB, int BS) {
  const int groups = n * HK * ((H / HK + 15) / 16);
  int64_t keys = (int64_t)NB * BS;
  if (window > 0 && window < keys) keys = window;
  if (chunk > 0 && chunk < keys) keys = chunk;
  const int steps = (int)((keys + 31) / 32);
  int s = 512 / (groups > 0 ? groups : 1);
  s = s < steps / 8 ? s : steps / 8;
  s = s < 32 ? s : 32;
  return s < 1 ? 1 : s;
}

template <int DKS, int VCB, int MAPS> int launch_rows(const RowsArgs& a, hipStream_t st) {
  const size_t smem = (((size_t)a.lds_pages * 4 + 15) & ~(size_t)15) + 4 * sizeof(float) * (16 * (a.V + 4) + 32);
  if (smem > 64 * 1024 &&
      hipFuncSetAttribute((const void*)grouped_rows_kernel<DKS, VCB, MAPS>, hipFuncAttributeMaxDynamicSharedMemorySize,
                          (int)smem) != hipSuccess) {
    zp_set_error("grouped_rows_attention: cannot reserve %zu bytes of LDS", smem);
    return ZP_EHIP;
  }
  hipLaunchKernelGGL((grouped_rows_kernel<DKS, VCB, MAPS>), dim3((unsigned)a.n * a.HK * a.htiles * a.splits), dim3(256), smem, st, a);
  ZP_LAUNCH_CHECK();
  if (a.splits > 1) {
    if (MAPS == 2) hipLaunchKernelGGL(grouped_pair_combine_kernel, dim3((unsigned)a.n * a.H / 2), dim3(64), 0, st, a);
    else hipLaunchKernelGGL(grouped_combine_kernel, dim3((unsigned)a.n * a.H), dim3(64), 0, st, a);
    ZP_LAUNCH_CHECK();
  }
  return ZP_OK;
}
template <int MAPS> int dispatch_rows(const RowsArgs& a, hipStream_t st) {
  const int dk = (a.D + 31) / 32;
  if (a.V <= 128) {
    if (dk <= 2) return launch_rows<2, 1, MAPS>(a, st);
    if (dk <= 4) return launch_rows<4, 1, MAPS>(a, st);
    return launch_rows<8, 1, MAPS>(a, st);
  }
  if (dk <= 4) return launch_rows<4, 2, MAPS>(a, st);
  return launch_rows<8, 2, MAPS>(a, st);
}

}  // namespace

extern "C" int zp_rotary_store(const void* in, const float* bias, const int32_t* positions, const float* freqs,
                               const zp_store_form* form, void* q_out, void* kv_out, void* cache, const int32_t* slots,
                               int32_t n, int32_t H, int32_t HK, int32_t D, int32_t VT, int32_t rot,
                               int64_t in_stride, int64_t num_slots, int32_t dtype, void* stream) {
  const zp_store_form plain = {}, f = form ? *form : plain;
  ZP_REQUIRE(n >= 0 && H > 0 && HK > 0 && D > 0 && VT > 0 && rot >= 0 && rot % 2 == 0 && rot <= D && num_slots > 0 &&
                 in_stride >= (int64_t)(H + HK) * D + (f.tied ? 0 : VT), "rotary_store: bad dims");
  ZP_MODEL_DTYPE("rotary_store");
  if (D % 8 != 0 || VT % 8 != 0 || in_stride % 8 != 0 || rot > 2048) {
    zp_set_error("rotary_store: head size %d, value columns %d (multiples of 8), %d rotated (<= 2048)", D, VT, rot);
    return ZP_EUNSUPPORTED;
  }
  if (n == 0) return ZP_OK;
  ZP_REQUIRE(in && positions && q_out && cache && slots && (rot == 0 || freqs), "rotary_store: null pointer");
  ZP_REQUIRE(aligned16(in) && aligned16(q_out) && aligned16(kv_out) && aligned16(cache) && aligned16(bias) && aligned16(f.norm),
             "rotary_store: tensors must be 16-byte aligned");
  ZP_REQUIRE(!f.norm || (!bias && f.q_norm > 0 && f.k_norm > 0), "rotary_store: norms of whole projections go without a bias");
  ZP_REQUIRE(!f.tied || !bias, "rotary_store: values that are the keys go without a bias");
  ZP_REQUIRE(!f.tied || VT == HK * D, "rotary_store: values that are the keys have their size");
  ZP_REQUIRE(!f.value_freqs || (f.turns && f.V > 0 && f.V % 8 == 0 && f.V <= 1024 && VT % f.V == 0),
             "rotary_store: values that turn need their head size and room for the turns");
  RotaryArgs a = {in, bias, positions, freqs, q_out, kv_out, cache, slots, n, H, HK, D, VT, rot / 2, in_stride, num_slots,
                  f.norm, f.q_norm, f.k_norm, f.eps, f.tied != 0, f.V, f.value_freqs, (float2*)f.turns};
  const int tokens = n < 2048 ? 1 : 4;
  const int64_t row = (int64_t)(H + HK) * D * zp_dtype_bytes(dtype);
  if (f.norm && row * tokens <= 32 * 1024) a.staged = (int)row;
  const unsigned grid = (unsigned)((n + tokens - 1) / tokens);
  const size_t smem = ((sizeof(float2) * tokens * (rot / 2 + (f.value_freqs ? f.V / 2 : 0)) + 15) & ~(size_t)15) + tokens * a.staged;
  hipStream_t st = (hipStream_t)stream;
  const bool norm = f.norm || f.tied, turn = f.value_freqs != nullptr;
  ZP_REQUIRE(smem <= 64 * 1024 && (int64_t)(H + HK) * D + VT < (1 << 24), "rotary_store: heads of %d, %d rotated: too long", D, rot);
#define ZP_ROTARY_FORM(T, VEC, N, NORM, TURN) \
  hipLaunchKernelGGL((rotary_store_kernel<T, VEC, N, NORM, TURN>), dim3(grid), dim3(256), smem, st, a)
#define ZP_ROTARY_N(T, VEC, N)                                     \
  do {                                                             \
    if (norm && turn) ZP_ROTARY_FORM(T, VEC, N, true, true);       \
    else if (norm) ZP_ROTARY_FORM(T, VEC, N, true, false);         \
    else if (turn) ZP_ROTARY_FORM(T, VEC, N, false, true);         \
    else ZP_ROTARY_FORM(T, VEC, N, false, false);                  \
  } while (0)
#define ZP_ROTARY(T, VEC)                                          \
  do {                                                             \
    if (tokens == 1) ZP_ROTARY_N(T, VEC, 1); else ZP_ROTARY_N(T, VEC, 4); \
  } while (0)
  if (dtype == ZP_BF16) {
    if (rot % 16 == 0) ZP_ROTARY(BF16, 8); else ZP_ROTARY(BF16, 1);
  } else {
    if (rot % 16 == 0) ZP_ROTARY(F32, 8); else ZP_ROTARY(F32, 1);
  }
#undef ZP_ROTARY
#undef ZP_ROTARY_N
#undef ZP_ROTARY_FORM
  ZP_LAUNCH_CHECK();
  return ZP_OK;
}

// D: length of a key head, all its maps together
static bool rows_need_plain(int D, int V, int BS, int dtype) {
  return dtype == ZP_F32 || D > 256 || V > 256 || BS < 16 || (BS & (BS - 1)) != 0;
}

extern "C" int64_t zp_grouped_rows_workspace(int32_t n, int32_t H, int32_t HK, int32_t D, int32_t V, int32_t maps,
                                             int32_t window, int32_t chunk, int32_t NB, int32_t BS,
                                             int32_t dtype) {
  if (n < 0 || H <= 0 || HK <= 0 || H % HK || V <= 0 || NB <= 0 || BS <= 0 || (maps != 1 && maps != 2)) return -1;
  if (rows_need_plain(D * maps, V, BS, dtype)) return 0;
  const int s = rows_splits(n, H * maps, HK, window, chunk, NB, BS);
  return s == 1 ? 0 : (int64_t)n * H * maps * s * (V + 2) * 4;
}

extern "C" int zp_grouped_rows_attention(const void* q, const void* cache, const int32_t* table,
                                         const int32_t* context_lens, const int32_t* table_rows,
                                         const float* sinks, const zp_attention_form* form, void* out, int32_t n,
                                         int32_t H, int32_t HK, int32_t D, int32_t V, int32_t BS, int32_t B,
                                         int32_t NB, int32_t num_pages, int32_t window, int32_t chunk,
                                         int64_t out_stride, float scale, float out_scale, int32_t dtype,
                                         void* workspace, int64_t workspace_bytes, void* stream) {
  const zp_attention_form plain = {0.f, 1, 0.f, 0.f, 0, nullptr, 0, nullptr}, f = form ? *form : plain;
  const bool two = f.maps == 2;
  ZP_REQUIRE(n >= 0 && H > 0 && HK > 0 && H % HK == 0 && D > 0 && V > 0 && BS > 0 && B > 0 && NB > 0 &&
                 num_pages > 0 && window >= 0 && chunk >= 0 && !(window && chunk) && (f.maps == 1 || two) &&
                 f.softcap >= 0.f, "grouped_rows_attention: bad dims");
  ZP_MODEL_DTYPE("grouped_rows_attention");
  if (D % 8 != 0 || V % 8 != 0 || V > 1024 || D > 4096) {
    zp_set_error("grouped_rows_attention: head sizes %d, %d unsupported (multiples of 8, <= 4096, <= 1024)", D, V);
    return ZP_EUNSUPPORTED;
  }
  if (n == 0) return ZP_OK;
  ZP_REQUIRE(q && cache && table && context_lens && out, "grouped_rows_attention: null pointer");
  ZP_REQUIRE(table_rows || n <= B, "grouped_rows_attention: more tokens than table rows");
  ZP_REQUIRE(!two || (!sinks && !f.turns && f.vdim > 0 && f.vdim <= V && (!f.gate || f.gate_stride >= (int64_t)H * V)),
             "grouped_rows_attention: two maps go without sinks and turns, with a mean over the values");
  ZP_REQUIRE(aligned16(q) && aligned16(cache) && aligned16(out) && aligned16(workspace) && aligned16(f.gate) &&
                 f.gate_stride % 8 == 0 && out_stride % 8 == 0 && out_stride >= (int64_t)H * V,
             "grouped_rows_attention: tensors must be 16-byte aligned");
  const int DK = D * f.maps;
  RowsArgs a = {};
  a.q = q; a.cache = cache; a.table = table; a.ctx = context_lens; a.seq = table_rows; a.sinks = sinks; a.out = out;
  a.part = (float*)workspace; a.n = n; a.H = H * f.maps; a.HK = HK; a.D = DK; a.V = V; a.BS = BS; a.B = B; a.NB = NB;
  a.num_pages = num_pages; a.window = window; a.chunk = chunk; a.o_st = out_stride; a.scale = scale;
  a.out_scale = out_scale; a.bs_shift = -1; a.cap = f.softcap; a.balance = f.balance; a.eps = f.eps; a.vdim = f.vdim;
  a.gate = f.gate; a.g_st = f.gate_stride; a.turns = (const float2*)f.turns;
  if ((BS & (BS - 1)) == 0)
    for (a.bs_shift = 0; (1 << a.bs_shift) < BS; ++a.bs_shift) {}
  int64_t pages = NB;
  const int seen = window > 0 ? window : chunk;
  if (seen > 0 && (seen - 1) / BS + 2 < pages) pages = (seen - 1) / BS + 2;
  hipStream_t st = (hipStream_t)stream;
  if (rows_need_plain(DK, V, BS, dtype) || pages > kMaxLdsPages) {
    const size_t smem = sizeof(float) * D;
    const dim3 grid((unsigned)n * H);
#define ZP_PLAIN(T)                                                                              \
  do {                                                                                           \
    if (two) hipLaunchKernelGGL((grouped_plain_kernel<T, 2>), grid, dim3(256), smem, st, a);     \
    else hipLaunchKernelGGL((grouped_plain_kernel<T, 1>), grid, dim3(256), smem, st, a);         \
  } while (0)
    if (dtype == ZP_BF16) ZP_PLAIN(BF16); else ZP_PLAIN(F32);
#undef ZP_PLAIN
    ZP_LAUNCH_CHECK();
    return ZP_OK;
  }
  a.htiles = (a.H / HK + 15) / 16;
  a.lds_pages = (int)pages;
  a.splits = rows_splits(n, a.H, HK, window, chunk, NB, BS);
  ZP_REQUIRE(a.splits == 1 || (workspace && workspace_bytes >= zp_grouped_rows_workspace(n, H, HK, D, V, f.maps, window, chunk, NB, BS, dtype)),
             "grouped_rows_attention: workspace too small");
  return two ? dispatch_rows<2>(a, st) : dispatch_rows<1>(a, st);
}
