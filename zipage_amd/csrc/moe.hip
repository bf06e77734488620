// Mixture of experts, without a host decision anywhere: every launch shape follows from the number of
// tokens, so a step can be captured into a graph.
//
//   small_linear     products with few outputs whose result stays in fp32 (router logits)
//   moe_select       softmax or sigmoids, the best groups of experts, the best experts of those
//   moe_plan         assignments in the order of their experts, and the list of row tiles
//   moe_gate_up      both input products of an expert for a row tile, its activation and the weight
//   moe_down         the output product; each assignment's row goes to the plane of its slot
//
// An assignment is (token n, slot j), written n * (top + 1) + j; slot `top` is the shared expert's,
// which every token uses with weight 1 and which counts as expert E.  Without a shared expert slots
// are 0 .. top - 1.
//
// Expert weights are kept in the order the matrix cores read them: [out / 16][in / step][lane][16
// bytes], where lane (g, r) holds row r and elements g * 16 bytes .. of a step of 64 bytes per row; a
// wave's operand is then one contiguous KB.  W is the row operand: a lane ends with four consecutive
// outputs of one token.
#include "mfma.h"

namespace {

template <typename T> struct Mma;
template <> struct Mma<BF16> {
  static constexpr int kStep = 32;
  __device__ static __forceinline__ f32x4 go(const u32x4& w, const u32x4& x, const f32x4& c) { return mfma_bf16(w, x, c); }
  __device__ static __forceinline__ void st4(void* p, int64_t i, const float* v) {
    uint2 o;
    o.x = pack_bf16(v[0], v[1]);
    o.y = pack_bf16(v[2], v[3]);
    *(uint2*)((uint16_t*)p + i) = o;
  }
};
template <> struct Mma<F32> {
  static constexpr int kStep = 16;
  __device__ static __forceinline__ f32x4 go(const u32x4& w, const u32x4& x, f32x4 c) {
    const f32x4 a = __builtin_bit_cast(f32x4, w), b = __builtin_bit_cast(f32x4, x);
#pragma unroll
    for (int j = 0; j < 4; ++j) c = __builtin_amdgcn_mfma_f32_16x16x4f32(a[j], b[j], c, 0, 0, 0);
    return c;
  }
  __device__ static __forceinline__ void st4(void* p, int64_t i, const float* v) {
    *(f32x4*)((float*)p + i) = f32x4{v[0], v[1], v[2], v[3]};
  }
};
template <typename T> constexpr int kPiece = 16 / T::bytes;   // elements a lane holds per step

// ------------------------------------------------------------------ few outputs, fp32
struct SmallArgs {
  const void* x;    // token rows of x_st elements
  const void* w;    // (M, K)
  float* out;       // (n, M)
  int n, K, M;
  int64_t x_st;
};

// 16 tokens x 16 * MT outputs per workgroup, its NW waves share the contraction.
template <typename T, int MT, int NW>
__global__ __launch_bounds__(64 * NW) void small_linear_kernel(SmallArgs a) {
  __shared__ float red[NW - 1][MT * 64 * 4];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l16 = lane & 15, g = lane >> 4;
  const int n0 = blockIdx.x * 16, m0 = blockIdx.y * 16 * MT;
  const int steps = a.K / Mma<T>::kStep;
  const char* x = (const char*)a.x + ((int64_t)min(n0 + l16, a.n - 1) * a.x_st + g * kPiece<T>) * T::bytes;
  const char* w[MT];
#pragma unroll
  for (int t = 0; t < MT; ++t)
    w[t] = (const char*)a.w + ((int64_t)min(m0 + t * 16 + l16, a.M - 1) * a.K + g * kPiece<T>) * T::bytes;
  f32x4 acc[MT];
#pragma unroll
  for (int t = 0; t < MT; ++t) acc[t] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
  for (int ks = wave; ks < steps; ks += NW) {
    const u32x4 xf = *(const u32x4*)(x + (int64_t)ks * 64);
#pragma unroll
    for (int t = 0; t < MT; ++t) acc[t] = Mma<T>::go(*(const u32x4*)(w[t] + (int64_t)ks * 64), xf, acc[t]);
  }
  if (wave > 0) {
#pragma unroll
    for (int t = 0; t < MT; ++t) *(f32x4*)(red[wave - 1] + (t * 64 + lane) * 4) = acc[t];
  }
  __syncthreads();
  if (wave > 0) return;
  const int n = n0 + l16;
#pragma unroll
  for (int t = 0; t < MT; ++t) {
#pragma unroll
    for (int k = 0; k < NW - 1; ++k) acc[t] += *(const f32x4*)(red[k] + (t * 64 + lane) * 4);
    const int m = m0 + t * 16 + g * 4;
    if (n < a.n && m < a.M) *(f32x4*)(a.out + (int64_t)n * a.M + m) = acc[t];
  }
}

// ------------------------------------------------------------------ selection
constexpr int kMaxExperts = 1024;

struct SelectArgs {
  const float* z;     // (n, z_st) router logits
  int32_t* ids;       // (n, top)
  float* weights;     // (n, top)
  int32_t* counts;    // (E + 1,), cleared here
  int n, E, top, groups, keep, score, z_st;
};

__device__ __forceinline__ int lowest_holder(float best, const float* v, int per) {
  // smallest index lane + 64 j whose value is `best`
  for (int j = 0; j < per; ++j) {
    const uint64_t b = __ballot(v[j] == best);
    if (b) return j * 64 + __builtin_ctzll(b);
  }
  return 0;
}

// A wave per token.  PER values per lane: expert (or group) lane + 64 j.
template <int PER>
__global__ __launch_bounds__(256) void moe_select_kernel(SelectArgs a) {
  extern __shared__ float lds[];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  if (blockIdx.x == 0)
    for (int e = threadIdx.x; e <= a.E; e += 256) a.counts[e] = 0;
  const int n = blockIdx.x * 4 + wave;
  float* const zl = lds + wave * a.E;
  float z[PER];
  float mx = -INFINITY;
  if (n < a.n) {
#pragma unroll
    for (int j = 0; j < PER; ++j) {
      const int e = lane + 64 * j;
      z[j] = e < a.E ? a.z[(int64_t)n * a.z_st + e] : -INFINITY;
      if (e < a.E) zl[e] = z[j];
      mx = fmaxf(mx, z[j]);
    }
  }
  __syncthreads();
  if (n >= a.n) return;
  mx = wave_max(mx);
  float sum = 0.f;
#pragma unroll
  for (int j = 0; j < PER; ++j) sum += expf(z[j] - mx);
  const float inv = 1.f / wave_sum(sum);
  const int gs = a.E / a.groups;
  if (a.keep < a.groups) {
    float gm[PER];
    uint32_t kept = 0;                          // bit j: group lane + 64 j
#pragma unroll
    for (int j = 0; j < PER; ++j) {
      const int gr = lane + 64 * j;
      gm[j] = -INFINITY;
      if (gr < a.groups)
        for (int i = 0; i < gs; ++i) gm[j] = fmaxf(gm[j], zl[gr * gs + i]);
    }
    for (int k = 0; k < a.keep; ++k) {
      float b = -INFINITY;
#pragma unroll
      for (int j = 0; j < PER; ++j) b = fmaxf(b, gm[j]);
      b = wave_max(b);
      const int gr = lowest_holder(b, gm, PER);
#pragma unroll
      for (int j = 0; j < PER; ++j)
        if (gr == lane + 64 * j) { gm[j] = -INFINITY; kept |= 1u << j; }
    }
    // experts of the other groups leave: group g's bit is in lane g % 64
#pragma unroll
    for (int j = 0; j < PER; ++j) {
      const int e = min(lane + 64 * j, a.E - 1), gr = e / gs;
      const uint32_t bits = (uint32_t)__shfl((int)kept, gr & 63);
      if (!((bits >> (gr >> 6)) & 1u)) z[j] = -INFINITY;
    }
  }
  for (int k = 0; k < a.top; ++k) {
    float b = -INFINITY;
#pragma unroll
    for (int j = 0; j < PER; ++j) b = fmaxf(b, z[j]);
    b = wave_max(b);
    const int e = lowest_holder(b, z, PER);
#pragma unroll
    for (int j = 0; j < PER; ++j)
      if (e == lane + 64 * j) z[j] = -INFINITY;
    if (lane == 0) {
      a.ids[(int64_t)n * a.top + k] = e;
      a.weights[(int64_t)n * a.top + k] = a.score == ZP_SCORE_SIGMOID ? 1.f / (1.f + expf(-b)) : expf(b - mx) * inv;
    }
  }
}

// ------------------------------------------------------------------ plan
struct PlanArgs {
  const int32_t* ids;     // (n, top)
  int32_t* counts;        // (E + 1,) zero before the first plan launch (large plans)
  int32_t* base;          // (blocks, E) large plans
  int32_t* offsets;       // (E + 2,)
  int32_t* sorted;        // (n * slots,) assignments by expert
  int32_t* tiles;         // (max_tiles, 4): expert, first position in `sorted`, rows, 0
  int32_t* ntiles;
  int n, E, top, shared, rows, max_tiles;   // rows: most rows per tile
};
constexpr int kPlanThreads = 1024;
constexpr int kPlanBlock = 4096;    // assignments per workgroup of a large plan

// Exclusive prefix sum of one value per thread over the workgroup.
__device__ __forceinline__ int block_prefix(int v, int* red) {
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int inc = wave_prefix_sum_incl(v);
  __syncthreads();
  if (lane == 63) red[wave] = inc;
  __syncthreads();
  int before = 0;
  for (int w = 0; w < wave; ++w) before += red[w];
  return before + inc - v;
}

// Offsets and tiles from the counts in LDS (E of them); the shared expert's rows follow the others'.
__device__ __forceinline__ void offsets_and_tiles(const PlanArgs& a, const int* counts, int* offsets, int* red) {
  const int e = threadIdx.x;
  int c = e < a.E ? counts[e] : (e == a.E && a.shared ? a.n : 0);
  int at = block_prefix(c, red);
  at = min(at, a.n * (a.top + a.shared));             // counters that were not cleared stay in bounds
  c = min(c, a.n * (a.top + a.shared) - at);
  const int t = (c + a.rows - 1) / a.rows;
  const int first = block_prefix(t, red);
  if (e <= a.E) {
    offsets[e] = at;
    for (int i = 0; i < t; ++i)
      if (first + i < a.max_tiles)
        *(int4*)(a.tiles + (int64_t)(first + i) * 4) = make_int4(e, at + i * a.rows, min(a.rows, c - i * a.rows), 0);
    if (e == a.E) *a.ntiles = min(first + t, a.max_tiles);
  }
  __syncthreads();
}

__global__ __launch_bounds__(kPlanThreads) void moe_plan_kernel(PlanArgs a) {
  __shared__ int counts[kMaxExperts], offsets[kMaxExperts + 1], red[kPlanThreads / 64];
  const int tid = threadIdx.x, total = a.n * a.top, slots = a.top + a.shared;
  counts[tid] = 0;
  __syncthreads();
  for (int i = tid; i < total; i += kPlanThreads) atomicAdd(&counts[min(max(a.ids[i], 0), a.E - 1)], 1);
  __syncthreads();
  offsets_and_tiles(a, counts, offsets, red);
  for (int i = tid; i < total; i += kPlanThreads) {
    const int e = min(max(a.ids[i], 0), a.E - 1);
    const int n = i / a.top;
    a.sorted[min(atomicAdd(&offsets[e], 1), total - 1)] = n * slots + i - n * a.top;
  }
  if (a.shared)
    for (int n = tid; n < a.n; n += kPlanThreads) a.sorted[total + n] = n * slots + a.top;
}

// Large plans in three launches: each workgroup's counts claim a place behind the counts of others;
// offsets and tiles; placement.
__global__ __launch_bounds__(kPlanThreads) void moe_count_kernel(PlanArgs a) {
  __shared__ int counts[kMaxExperts];
  const int tid = threadIdx.x, total = a.n * a.top, i0 = blockIdx.x * kPlanBlock;
  counts[tid] = 0;
  __syncthreads();
  for (int i = i0 + tid; i < min(i0 + kPlanBlock, total); i += kPlanThreads)
    atomicAdd(&counts[min(max(a.ids[i], 0), a.E - 1)], 1);
  __syncthreads();
  if (tid < a.E) a.base[(int64_t)blockIdx.x * a.E + tid] = atomicAdd(&a.counts[tid], counts[tid]);
}
__global__ __launch_bounds__(kPlanThreads) void moe_offsets_kernel(PlanArgs a) {
  __shared__ int counts[kMaxExperts], offsets[kMaxExperts + 1], red[kPlanThreads / 64];
  const int tid = threadIdx.x;
  counts[tid] = tid < a.E ? a.counts[tid] : 0;
  __syncthreads();
  offsets_and_tiles(a, counts, offsets, red);
  for (int e = tid; e <= a.E; e += kPlanThreads) a.offsets[e] = offsets[e];
}
__global__ __launch_bounds__(kPlanThreads) void moe_place_kernel(PlanArgs a) {
  __shared__ int at[kMaxExperts];
  const int tid = threadIdx.x, total = a.n * a.top, i0 = blockIdx.x * kPlanBlock, slots = a.top + a.shared;
  if (tid < a.E) at[tid] = a.offsets[tid] + a.base[(int64_t)blockIdx.x * a.E + tid];
  __syncthreads();
  for (int i = i0 + tid; i < min(i0 + kPlanBlock, total); i += kPlanThreads) {
    const int n = i / a.top;
    a.sorted[min(atomicAdd(&at[min(max(a.ids[i], 0), a.E - 1)], 1), total - 1)] = n * slots + i - n * a.top;
  }
  if (a.shared)
    for (int n = blockIdx.x * kPlanThreads + tid; n < a.n; n += gridDim.x * kPlanThreads)
      a.sorted[total + n] = n * slots + a.top;
}

// ------------------------------------------------------------------ expert products
struct ExpertArgs {
  const void* x;          // gate_up: (n, K) tokens; down: (n * slots, K) rows by position in `sorted`
  const void* w;          // routed experts, back to back
  const void* w_shared;
  void* out;              // gate_up: (n * slots, o_st); down: planes (slots, n, o_st)
  const int32_t* sorted;
  const int32_t* tiles;
  const int32_t* ntiles;
  const float* weights;   // (n, top)
  int n, E, top, slots, max_tiles;
  int K, K_shared;        // contraction, routed and shared
  int M, M_shared;        // outputs (gate_up: of the gate alone)
  int64_t x_st, o_st, w_expert;   // w_expert: elements between experts
  int act;
  float limit, limit_shared;
};

// ZP_GATE_CLAMPED: w g sigmoid(1.702 g) (u + 1), g = min(gate, limit), u = clamp(up, -limit, limit)
// ZP_GATE_SILU: g sigmoid(g) u of the weighted products
template <typename T> __device__ __forceinline__ float gated(int act, float w, float gate, float up, float limit) {
  if (act == ZP_GATE_SILU) {
    const float g = w * gate;
    return g * sigmoid_of<T>(g) * (w * up);
  }
  const float g = fminf(gate, limit), u = fminf(fmaxf(up, -limit), limit);
  return w * (g * sigmoid_of<T>(1.702f * g) * (u + 1.f));
}

// Few rows per expert: the weights are streamed straight into registers.  A workgroup owns 64 rows of W (gate_up:
// two 16-row tiles of the gate and the two of `up` that belong to them) and up to 16 * MT tokens; its four waves
// take every fourth step of the contraction and meet in LDS.
constexpr int kRowsW = 4;                              // 16-row tiles of W
template <typename T, int MT, bool UP>
__global__ __launch_bounds__(256) void expert_rows_kernel(ExpertArgs a) {
  __shared__ __align__(16) float part[4][kRowsW * MT * 256];
  const int lane = threadIdx.x & 63, l16 = lane & 15, g = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int tile = blockIdx.x % a.max_tiles, cb = blockIdx.x / a.max_tiles;
  if (tile >= *a.ntiles) return;
  const int4 t = *(const int4*)(a.tiles + (int64_t)tile * 4);
  const bool shared = t.x == a.E;
  const int wtiles = (shared ? a.M_shared : a.M) / 16 * (UP ? 2 : 1), K = shared ? a.K_shared : a.K;
  const int w0 = cb * kRowsW;
  if (w0 >= wtiles) return;
  const int steps = K / Mma<T>::kStep;
  const char* const w = (const char*)(shared ? a.w_shared : a.w) + (shared ? 0 : t.x * a.w_expert) * T::bytes + lane * 16;
  const char* wp[kRowsW];
#pragma unroll
  for (int i = 0; i < kRowsW; ++i) wp[i] = w + (int64_t)min(w0 + i, wtiles - 1) * steps * 1024;
  const char* x[MT];
#pragma unroll
  for (int i = 0; i < MT; ++i) {
    const int pos = t.y + min(i * 16 + l16, t.z - 1);
    const int64_t row = UP ? a.sorted[pos] / a.slots : pos;
    x[i] = (const char*)a.x + (row * a.x_st + g * kPiece<T>) * T::bytes;
  }
  f32x4 acc[kRowsW][MT];
#pragma unroll
  for (int k = 0; k < kRowsW; ++k)
#pragma unroll
    for (int i = 0; i < MT; ++i) acc[k][i] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
  for (int ks = wave; ks < steps; ks += 4) {
    u32x4 wf[kRowsW], xf[MT];
#pragma unroll
    for (int k = 0; k < kRowsW; ++k) {
      const u32x4* const p = (const u32x4*)(wp[k] + (int64_t)ks * 1024);
      if constexpr (MT == 1) wf[k] = __builtin_nontemporal_load(p);       // hardly any expert has a second tile
      else wf[k] = *p;
    }
#pragma unroll
    for (int i = 0; i < MT; ++i) xf[i] = *(const u32x4*)(x[i] + (int64_t)ks * 64);
#pragma unroll
    for (int k = 0; k < kRowsW; ++k)
#pragma unroll
      for (int i = 0; i < MT; ++i) acc[k][i] = Mma<T>::go(wf[k], xf[i], acc[k][i]);
  }
#pragma unroll
  for (int k = 0; k < kRowsW; ++k)
#pragma unroll
    for (int i = 0; i < MT; ++i) *(f32x4*)(part[wave] + ((k * MT + i) * 64 + lane) * 4) = acc[k][i];
  __syncthreads();
  auto total = [&](int k, int i) {
    f32x4 r = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int v = 0; v < 4; ++v) r += *(const f32x4*)(part[v] + ((k * MT + i) * 64 + lane) * 4);
    return r;
  };
  for (int u = wave; u < (UP ? kRowsW / 2 : kRowsW) * MT; u += 4) {
    const int i = u % MT, k = u / MT * (UP ? 2 : 1), wt = w0 + k;
    if (wt >= wtiles || i * 16 + l16 >= t.z) continue;
    const int pos = t.y + i * 16 + l16, as = a.sorted[pos], n = as / a.slots, slot = as - n * a.slots;
    const f32x4 first = total(k, i);
    float r[4];
    if constexpr (UP) {
      const f32x4 second = total(k + 1, i);
      const float wgt = slot < a.top ? a.weights[(int64_t)n * a.top + slot] : 1.f;
      const float lim = shared ? a.limit_shared : a.limit;
#pragma unroll
      for (int e = 0; e < 4; ++e) r[e] = gated<T>(a.act, wgt, first[e], second[e], lim);
      Mma<T>::st4(a.out, (int64_t)pos * a.o_st + wt * 8 + g * 4, r);
    } else {
#pragma unroll
      for (int e = 0; e < 4; ++e) r[e] = first[e];
      Mma<T>::st4(a.out, ((int64_t)slot * a.n + n) * a.o_st + wt * 16 + g * 4, r);
    }
  }
}

// Many rows per expert: 128 tokens x 256 rows of W per workgroup, both streamed straight into LDS in the
// order the matrix cores read them, 32 of the contraction at a time, two stages ahead of the products; one
// barrier per stage.  A wave owns 64 tokens x 128 rows of W.
typedef __attribute__((address_space(3))) void* lds_ptr_t;
constexpr int kBlockRows = 128;                        // tokens
constexpr int kBlockW = 16;                            // 16-row tiles of W
constexpr int kStageBytes = (kBlockRows / 16 + kBlockW) * 1024, kStages = 3;

template <bool UP>
__global__ __launch_bounds__(256, 2) void expert_tiles_kernel(ExpertArgs a) {
  extern __shared__ __align__(16) char lds_raw[];
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), l16 = lane & 15, g = lane >> 4;
  // An XCD takes a contiguous share of the (tile, column block) pairs, in squares of eight by eight, so that
  // what is in flight on it shares rows of x and of W in its L2.
  const int nt = *a.ntiles;
  const int Mx = max(a.M, a.M_shared) * (UP ? 2 : 1), cols = (Mx + 16 * kBlockW - 1) / (16 * kBlockW);
  const int groups = (nt + 7) / 8, i_xcd = blockIdx.x >> 3;
  if (i_xcd >= groups * cols) return;
  const int lin = (blockIdx.x & 7) * groups * cols + i_xcd;
  const int tg = lin / (8 * cols), rem = lin - tg * 8 * cols;
  const int tile = tg * 8 + (rem & 7), cb = rem >> 3;
  if (tile >= nt) return;
  const int4 t = *(const int4*)(a.tiles + (int64_t)tile * 4);
  const bool shared = t.x == a.E;
  const int wtiles = (shared ? a.M_shared : a.M) / 16 * (UP ? 2 : 1), K = shared ? a.K_shared : a.K;
  const int w0 = cb * kBlockW;
  if (w0 >= wtiles) return;
  const int steps = K / 32;
  const char* wbase = (const char*)(shared ? a.w_shared : a.w) + (shared ? 0 : t.x * a.w_expert) * 2;
  const __amdgpu_buffer_rsrc_t rw = __builtin_amdgcn_make_buffer_rsrc((void*)(wbase + (int64_t)w0 * steps * 1024), 0,
                                                                      min(kBlockW, wtiles - w0) * steps * 1024, 0x00020000);
  // gate_up gathers tokens from all of x, down reads consecutive rows
  const char* const xbase = (const char*)a.x + (UP ? 0 : t.y * a.x_st * 2);
  const __amdgpu_buffer_rsrc_t rx = __builtin_amdgcn_make_buffer_rsrc((void*)xbase, 0, (int)((UP ? a.n : t.z) * a.x_st * 2), 0x00020000);
  // this wave's loads of a stage: two of the eight 16-token tiles, four of the sixteen of W
  int xoff[2], woff[4];
#pragma unroll
  for (int i = 0; i < 2; ++i) {
    const int r = min((wave * 2 + i) * 16 + l16, t.z - 1);
    xoff[i] = (int)((UP ? a.sorted[t.y + r] / a.slots : r) * a.x_st * 2) + g * 16;
  }
#pragma unroll
  for (int i = 0; i < 4; ++i) woff[i] = min(wave * 4 + i, wtiles - w0 - 1) * steps * 1024;
  auto request = [&](int ks) {
    char* const st = lds_raw + (ks % kStages) * kStageBytes;
#pragma unroll
    for (int i = 0; i < 2; ++i)
      __builtin_amdgcn_raw_ptr_buffer_load_lds(rx, (lds_ptr_t)(st + (wave * 2 + i) * 1024), 16, xoff[i], ks * 64, 0, 0);
#pragma unroll
    for (int i = 0; i < 4; ++i)
      __builtin_amdgcn_raw_ptr_buffer_load_lds(rw, (lds_ptr_t)(st + (8 + wave * 4 + i) * 1024), 16, lane * 16,
                                               woff[i] + ks * 1024, 0, 0);
  };
  const int th = wave & 1, wh = wave >> 1;
  f32x4 acc[8][4];
#pragma unroll
  for (int i = 0; i < 8; ++i)
#pragma unroll
    for (int j = 0; j < 4; ++j) acc[i][j] = f32x4{0.f, 0.f, 0.f, 0.f};
  request(0);
  if (steps > 1) request(1);
#pragma unroll 1
  for (int ks = 0; ks < steps; ++ks) {
    if (ks + 1 < steps) asm volatile("s_waitcnt vmcnt(6)" ::: "memory");
    else asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    __builtin_amdgcn_s_barrier();                        // everyone's part of the stage is there
    if (ks + 2 < steps) request(ks + 2);                 // over the stage that was used up before the barrier
    const char* const st = lds_raw + (ks % kStages) * kStageBytes + lane * 16;
    u32x4 xf[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) xf[j] = *(const u32x4*)(st + (th * 4 + j) * 1024);
    u32x4 wf[8];
#pragma unroll
    for (int i = 0; i < 8; ++i) wf[i] = *(const u32x4*)(st + (8 + wh * 8 + i) * 1024);
    __builtin_amdgcn_sched_barrier(0);                   // all reads on their way before the first product
#pragma unroll
    for (int i = 0; i < 8; ++i)
#pragma unroll
      for (int j = 0; j < 4; ++j) acc[i][j] = mfma_bf16(wf[i], xf[j], acc[i][j]);
    __builtin_amdgcn_sched_barrier(0);
  }
  // Two result tiles side by side hold 4 outputs per lane each; lanes of neighbouring groups swap halves, so that
  // each ends with 8 consecutive outputs of one of them: group g has tile (g & 1), outputs 8 (g >> 1) on.
  auto store8 = [&](const float* lo, const float* hi, int64_t at, int tile, int tiles, bool row) {
    const auto a0 = __builtin_amdgcn_permlane16_swap(pack_bf16(lo[0], lo[1]), pack_bf16(hi[0], hi[1]), false, false);
    const auto a1 = __builtin_amdgcn_permlane16_swap(pack_bf16(lo[2], lo[3]), pack_bf16(hi[2], hi[3]), false, false);
    if (row && tile + (g & 1) < tiles)
      *(u32x4*)((uint16_t*)a.out + at + (tile + (g & 1)) * 16 + (g >> 1) * 8) = u32x4{a0[0], a1[0], a0[1], a1[1]};
  };
  const int out_tiles = UP ? wtiles / 2 : wtiles;
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    const int r = (th * 4 + j) * 16 + l16;
    const bool row = r < t.z;                          // every lane takes part in the swaps
    const int pos = t.y + min(r, t.z - 1), as = a.sorted[pos], n = as / a.slots, slot = as - n * a.slots;
    if constexpr (UP) {
      const float wgt = slot < a.top ? a.weights[(int64_t)n * a.top + slot] : 1.f;
      const float lim = shared ? a.limit_shared : a.limit;
#pragma unroll
      for (int i = 0; i < 8; i += 4) {
        float v[2][4];
#pragma unroll
        for (int u = 0; u < 2; ++u)
#pragma unroll
          for (int k = 0; k < 4; ++k) v[u][k] = gated<BF16>(a.act, wgt, acc[i + 2 * u][j][k], acc[i + 2 * u + 1][j][k], lim);
        store8(v[0], v[1], (int64_t)pos * a.o_st, (w0 + wh * 8 + i) / 2, out_tiles, row);
      }
    } else {
#pragma unroll
      for (int i = 0; i < 8; i += 2) {
        const float lo[4] = {acc[i][j][0], acc[i][j][1], acc[i][j][2], acc[i][j][3]};
        const float hi[4] = {acc[i + 1][j][0], acc[i + 1][j][1], acc[i + 1][j][2], acc[i + 1][j][3]};
        store8(lo, hi, ((int64_t)slot * a.n + n) * a.o_st, w0 + wh * 8 + i, out_tiles, row);
      }
    }
  }
}

template <bool UP> int launch_experts(const ExpertArgs& a, int rows, int dtype, hipStream_t st) {
  if (rows == kBlockRows) {
    const int Mx = (a.M > a.M_shared ? a.M : a.M_shared) * (UP ? 2 : 1);
    const int64_t grid = (int64_t)((a.max_tiles + 7) / 8) * 8 * ((Mx + 16 * kBlockW - 1) / (16 * kBlockW));
    constexpr int smem = kStages * kStageBytes;
    if (hipFuncSetAttribute((const void*)expert_tiles_kernel<UP>, hipFuncAttributeMaxDynamicSharedMemorySize, smem) != hipSuccess) {
      zp_set_error("moe: cannot reserve %d bytes of LDS", smem);
      return ZP_EHIP;
    }
    hipLaunchKernelGGL((expert_tiles_kernel<UP>), dim3((unsigned)grid), dim3(256), smem, st, a);
    ZP_LAUNCH_CHECK();
    return ZP_OK;
  }
  const int Mw = (a.M > a.M_shared ? a.M : a.M_shared) * (UP ? 2 : 1);
  const int64_t grid = (int64_t)a.max_tiles * ((Mw + 16 * kRowsW - 1) / (16 * kRowsW));
  if (grid >= (1ll << 31)) {
    zp_set_error("moe: too many tiles");
    return ZP_EUNSUPPORTED;
  }
#define ZP_EXPERTS(T, MT) hipLaunchKernelGGL((expert_rows_kernel<T, MT, UP>), dim3((unsigned)grid), dim3(256), 0, st, a)
#define ZP_EXPERT_ROWS(T)                 \
  do {                                    \
    if (rows == 16) ZP_EXPERTS(T, 1);     \
    else if (rows == 32) ZP_EXPERTS(T, 2);\
    else ZP_EXPERTS(T, 4);                \
  } while (0)
  if (dtype == ZP_BF16) ZP_EXPERT_ROWS(BF16); else ZP_EXPERT_ROWS(F32);
#undef ZP_EXPERT_ROWS
#undef ZP_EXPERTS
  ZP_LAUNCH_CHECK();
  return ZP_OK;
}

// Rows per tile: enough for the average expert.
int tile_rows(int n, int E, int top, int dtype) {
  const int64_t avg = ((int64_t)n * top + E - 1) / E;
  if (dtype == ZP_BF16 && avg > 48) return kBlockRows;
  return avg <= 8 ? 16 : (avg <= 16 ? 32 : 64);       // a second tile reads an expert's weights again
}
int tile_bound(int n, int E, int top, int shared, int rows) {
  const int64_t a = (int64_t)n * top;
  const int64_t used = a < E ? a : E;
  return (int)(a / rows + used + (shared ? (n + rows - 1) / rows : 0));
}

}  // namespace

extern "C" int zp_small_linear(const void* x, const void* w, float* out, int32_t n, int32_t K, int32_t M,
                               int64_t x_stride, int32_t dtype, void* stream) {
  ZP_REQUIRE(n >= 0 && K > 0 && M > 0 && x_stride >= K, "small_linear: bad dims");
  ZP_MODEL_DTYPE("small_linear");
  if (K % 32 != 0 || M % 4 != 0 || x_stride % 8 != 0) {
    zp_set_error("small_linear: K %d, M %d unsupported (multiples of 32 and 4)", K, M);
    return ZP_EUNSUPPORTED;
  }
  if (n == 0) return ZP_OK;
  ZP_REQUIRE(x && w && out && aligned16(x) && aligned16(w) && aligned16(out), "small_linear: null or unaligned pointer");
  SmallArgs a = {x, w, out, n, K, M, x_stride};
  hipStream_t st = (hipStream_t)stream;
  const unsigned gx = (unsigned)((n + 15) / 16);
  const bool wide = gx >= 256 && M > 16;
  const dim3 grid(gx, (unsigned)(wide ? (M + 63) / 64 : (M + 15) / 16));
#define ZP_SMALL(T)                                                                              \
  do {                                                                                           \
    if (wide) hipLaunchKernelGGL((small_linear_kernel<T, 4, 4>), grid, dim3(256), 0, st, a);     \
    else hipLaunchKernelGGL((small_linear_kernel<T, 1, 16>), grid, dim3(1024), 0, st, a);        \
  } while (0)
  if (dtype == ZP_BF16) ZP_SMALL(BF16); else ZP_SMALL(F32);
#undef ZP_SMALL
  ZP_LAUNCH_CHECK();
  return ZP_OK;
}

extern "C" int zp_moe_select(const float* logits, int32_t* ids, float* weights, int32_t* counts, int32_t n,
                             int32_t E, int32_t top, int32_t groups, int32_t keep, int32_t score,
                             int32_t logits_stride, void* stream) {
  ZP_REQUIRE(n >= 0 && E > 0 && top > 0 && groups > 0 && E % groups == 0 && keep > 0 && keep <= groups &&
                 top <= E / groups * keep && logits_stride >= E &&
                 (score == ZP_SCORE_SOFTMAX || score == ZP_SCORE_SIGMOID), "moe_select: bad dims");
  if (E > kMaxExperts - 1) {
    zp_set_error("moe_select: %d experts (at most %d)", E, kMaxExperts - 1);
    return ZP_EUNSUPPORTED;
  }
  if (n == 0) return ZP_OK;
  ZP_REQUIRE(logits && ids && weights && counts, "moe_select: null pointer");
  SelectArgs a = {logits, ids, weights, counts, n, E, top, groups, keep, score, logits_stride};
  const dim3 grid((unsigned)((n + 3) / 4));
  const size_t smem = sizeof(float) * 4 * E;
  hipStream_t st = (hipStream_t)stream;
  if (E <= 64) hipLaunchKernelGGL((moe_select_kernel<1>), grid, dim3(256), smem, st, a);
  else if (E <= 256) hipLaunchKernelGGL((moe_select_kernel<4>), grid, dim3(256), smem, st, a);
  else hipLaunchKernelGGL((moe_select_kernel<16>), grid, dim3(256), smem, st, a);
  ZP_LAUNCH_CHECK();
  return ZP_OK;
}

extern "C" int64_t zp_moe_tile_rows(int32_t n, int32_t E, int32_t top, int32_t dtype) {
  return n <= 0 || E <= 0 || top <= 0 ? -1 : tile_rows(n, E, top, dtype);
}
extern "C" int64_t zp_moe_max_tiles(int32_t n, int32_t E, int32_t top, int32_t shared, int32_t rows) {
  return n <= 0 || E <= 0 || top <= 0 || rows <= 0 ? -1 : tile_bound(n, E, top, shared, rows);
}
extern "C" int64_t zp_moe_plan_workspace(int32_t n, int32_t E, int32_t top) {
  if (n <= 0 || E <= 0 || top <= 0) return -1;
  return ((int64_t)(((int64_t)n * top + kPlanBlock - 1) / kPlanBlock) * E + E + 2) * 4;
}

extern "C" int zp_moe_plan(const int32_t* ids, int32_t* counts, int32_t* sorted, int32_t* tiles, int32_t* ntiles,
                           int32_t n, int32_t E, int32_t top, int32_t shared, int32_t rows, int32_t max_tiles,
                           void* workspace, int64_t workspace_bytes, void* stream) {
  ZP_REQUIRE(n > 0 && E > 0 && E < kMaxExperts && top > 0 && rows > 0 && (shared == 0 || shared == 1) &&
                 max_tiles >= tile_bound(n, E, top, shared, rows), "moe_plan: bad dims");
  ZP_REQUIRE(ids && counts && sorted && tiles && ntiles && aligned16(tiles), "moe_plan: null or unaligned pointer");
  ZP_REQUIRE((int64_t)n * (top + shared) < (1ll << 31), "moe_plan: too many tokens");
  PlanArgs a = {ids, counts, nullptr, nullptr, sorted, tiles, ntiles, n, E, top, shared, rows, max_tiles};
  hipStream_t st = (hipStream_t)stream;
  if ((int64_t)n * top <= 2 * kPlanBlock) {
    hipLaunchKernelGGL(moe_plan_kernel, dim3(1), dim3(kPlanThreads), 0, st, a);
    ZP_LAUNCH_CHECK();
    return ZP_OK;
  }
  ZP_REQUIRE(workspace && workspace_bytes >= zp_moe_plan_workspace(n, E, top), "moe_plan: workspace too small");
  a.offsets = (int32_t*)workspace;
  a.base = a.offsets + E + 2;
  const unsigned blocks = (unsigned)(((int64_t)n * top + kPlanBlock - 1) / kPlanBlock);
  hipLaunchKernelGGL(moe_count_kernel, dim3(blocks), dim3(kPlanThreads), 0, st, a);
  hipLaunchKernelGGL(moe_offsets_kernel, dim3(1), dim3(kPlanThreads), 0, st, a);
  hipLaunchKernelGGL(moe_place_kernel, dim3(blocks), dim3(kPlanThreads), 0, st, a);
  ZP_LAUNCH_CHECK();
  return ZP_OK;
}

static int experts(bool up, const void* x, const void* w, const void* w_shared, void* out, const int32_t* sorted,
                   const int32_t* tiles, const int32_t* ntiles, const float* weights, int32_t n, int32_t E,
                   int32_t top, int32_t shared, int32_t rows, int32_t max_tiles, int32_t K, int32_t K_shared,
                   int32_t M, int32_t M_shared, int64_t x_stride, int64_t out_stride, int32_t act,
                   float limit, float limit_shared, int32_t dtype, void* stream) {
  ZP_REQUIRE((act == ZP_GATE_CLAMPED || act == ZP_GATE_SILU) && n >= 0 && E > 0 && top > 0 && max_tiles > 0 && K > 0 && M > 0 && (!shared || (K_shared > 0 && M_shared > 0)),
             "moe experts: bad dims");
  ZP_MODEL_DTYPE("moe experts");
  if (K % 32 || K_shared % 32 || M % 16 || M_shared % 16 || x_stride % 8 || out_stride % 8 ||
      (rows != 16 && rows != 32 && rows != 64 && (rows != kBlockRows || dtype != ZP_BF16))) {
    zp_set_error("moe experts: sizes %d x %d, shared %d x %d, %d rows per tile unsupported", M, K, M_shared, K_shared, rows);
    return ZP_EUNSUPPORTED;
  }
  if (n == 0) return ZP_OK;
  ZP_REQUIRE(x && w && (!shared || w_shared) && out && sorted && tiles && ntiles && (!up || weights), "moe experts: null pointer");
  ZP_REQUIRE(aligned16(x) && aligned16(w) && aligned16(w_shared) && aligned16(out) && aligned16(tiles) &&
                 x_stride >= (K > K_shared ? K : K_shared) && out_stride >= (M > M_shared ? M : M_shared),
             "moe experts: unaligned or overlapping rows");
  if (rows == kBlockRows) {       // 31-bit byte offsets into x and into a block of W
    const int64_t xr = up ? n : kBlockRows, kx = K > K_shared ? K : K_shared;
    if (xr * x_stride * 2 >= (1ll << 31) || kx * 512 >= (1ll << 31)) {
      zp_set_error("moe experts: %lld rows of %lld elements in one step", (long long)xr, (long long)x_stride);
      return ZP_EUNSUPPORTED;
    }
  }
  ExpertArgs a = {x, w, w_shared, out, sorted, tiles, ntiles, weights, n, E, top, top + shared, max_tiles, K, K_shared,
                  M, shared ? M_shared : 0, x_stride, out_stride, (int64_t)M * K * (up ? 2 : 1), act, limit, limit_shared};
  return up ? launch_experts<true>(a, rows, dtype, (hipStream_t)stream)
            : launch_experts<false>(a, rows, dtype, (hipStream_t)stream);
}

extern "C" int zp_moe_gate_up(const void* x, const void* w, const void* w_shared, void* out, const int32_t* sorted,
                              const int32_t* tiles, const int32_t* ntiles, const float* weights, int32_t n,
                              int32_t E, int32_t top, int32_t shared, int32_t rows, int32_t max_tiles, int32_t K,
                              int32_t M, int32_t M_shared, int64_t x_stride, int64_t out_stride, int32_t act,
                              float limit, float limit_shared, int32_t dtype, void* stream) {
  return experts(true, x, w, w_shared, out, sorted, tiles, ntiles, weights, n, E, top, shared, rows, max_tiles, K, K,
                 M, M_shared, x_stride, out_stride, act, limit, limit_shared, dtype, stream);
}
extern "C" int zp_moe_down(const void* x, const void* w, const void* w_shared, void* out, const int32_t* sorted,
                           const int32_t* tiles, const int32_t* ntiles, int32_t n, int32_t E, int32_t top,
                           int32_t shared, int32_t rows, int32_t max_tiles, int32_t K, int32_t K_shared, int32_t M,
                           int64_t x_stride, int64_t out_stride, int32_t dtype, void* stream) {
  return experts(false, x, w, w_shared, out, sorted, tiles, ntiles, nullptr, n, E, top, shared, rows, max_tiles, K,
                 K_shared, M, M, x_stride, out_stride, ZP_GATE_CLAMPED, 0.f, 0.f, dtype, stream);
}
