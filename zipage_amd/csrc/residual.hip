// Row kernels of decoders that keep their residual stream in fp32 whatever the dtype of their
// matrix products: token + learned-position embedding, residual add (of branch outputs as they are or
// normed), depth average over all earlier layer results, RMS norm or tanh norm, the xIELU, squared relu
// and normed-powers activations, and the soft cap of logits.  Each is one pass over its rows (HBM- or
// launch-bound): the stream is read once, and what the next matrix product needs leaves the same
// launch in that product's dtype.
#include "models.h"
#include <math.h>

namespace {

constexpr int kMaxPieces = 4;   // 8-element pieces per thread: rows up to 8 * 4 * 256 elements
constexpr int kMaxBranches = 3, kMaxNormed = 2;

// A branch output that joins the stream: the sum of n planes of (rows, width) T.
struct Branch {
  const void* y;
  const float* w;         // (width,) weight of an RMS norm on the sum before it joins, or null
  int n;
};

struct RowArgs {
  // source: an embedding (tokens, positions) or the stream x plus branch outputs, those with a norm first
  const int64_t* tokens;
  const int32_t* positions;
  const void* embed;      // (vocab, width) T
  const void* pos;        // (max_positions, width) T or null
  int64_t vocab, max_positions;
  const float* x;         // (n, width) fp32
  Branch br[kMaxBranches];
  int n_br;
  int64_t y_plane;        // elements between a branch's planes
  float embed_scale;
  // depth average: result_new = sum_j mix[j] * hist[j] + mix[n_hist] * (x + branches)
  const float* hist;      // n_hist planes of (n, width) fp32
  int64_t hist_plane;     // elements between planes
  const float* mix;       // n_hist + 1 weights, or null: the sum itself goes on
  int n_hist;
  const float* shift;     // (width,) added to every row after the average, or null
  float* result;          // receives the embedding, or x + branches, before average and shift; or null
  float* x_out;           // receives what goes on, or null
  const float* w;         // (width,) norm weight, or null: no norm
  const float* b;         // (width,) tanh norm: tanh(alpha x) * (offset + w) + b; null: RMS norm
  void* out;              // (n, width) T: norm(x_out) * (offset + w) * out_scale
  int width, norm_width;  // padded row length, and the length the mean is taken over
  float eps, offset, out_scale, alpha;
};

// One workgroup of THREADS per row; the row lives in registers.
template <int kW> __device__ __forceinline__ float row_sum(float v, float* red, int tid) {
  v = wave_sum(v);
  if (kW > 1) {
    if ((tid & 63) == 0) red[tid >> 6] = v;
    __syncthreads();
    v = 0.f;
#pragma unroll
    for (int i = 0; i < kW; ++i) v += red[i];
  }
  return v;
}

// One piece of a branch: the sum of its planes.
template <typename T> __device__ __forceinline__ void branch_sum(const Branch& b, int64_t plane, int64_t at, float* y) {
  Vec8<T>::ld(b.y, at, y);
  int j = 1;
  for (; j + 4 <= b.n; j += 4) {
    float r[4][8];
#pragma unroll
    for (int u = 0; u < 4; ++u) Vec8<T>::ld(b.y, (j + u) * plane + at, r[u]);
#pragma unroll
    for (int u = 0; u < 4; ++u)
#pragma unroll
      for (int i = 0; i < 8; ++i) y[i] += r[u][i];
  }
  for (; j < b.n; ++j) {
    float r[8];
    Vec8<T>::ld(b.y, j * plane + at, r);
#pragma unroll
    for (int i = 0; i < 8; ++i) y[i] += r[i];
  }
}

// NORMED: so many branches are normed before they join.
template <typename T, int THREADS, bool EMBED, int NORMED>
__global__ __launch_bounds__(THREADS) void row_kernel(RowArgs a) {
  constexpr int kW = THREADS / 64, NB = NORMED > 0 ? NORMED : 1;
  __shared__ float red[kW], red_y[NB][kW];
  const int tid = threadIdx.x;
  const int64_t row = blockIdx.x;
  const int pieces = a.width / 8;
  float v[kMaxPieces][8];
  float ss = 0.f;
  float y[NB][NORMED > 0 ? kMaxPieces : 1][8];     // the normed branches: their sums first, the stream joins later
  float ry[NB];
  if constexpr (NORMED > 0) {
#pragma unroll
    for (int b = 0; b < NB; ++b) {
      ry[b] = 0.f;
#pragma unroll
      for (int k = 0; k < kMaxPieces; ++k) {
        const int pc = tid + k * THREADS;
        if (pc < pieces) {
          branch_sum<T>(a.br[b], a.y_plane, row * a.width + pc * 8, y[b][k]);
#pragma unroll
          for (int i = 0; i < 8; ++i) ry[b] += y[b][k][i] * y[b][k][i];
        }
      }
    }
#pragma unroll
    for (int b = 0; b < NB; ++b) ry[b] = 1.f / sqrtf(row_sum<kW>(ry[b], red_y[b], tid) / (float)a.norm_width + a.eps);
  }
  int64_t tok = 0, ps = 0;
  if (EMBED) {
    tok = a.tokens[row];
    tok = tok < 0 ? 0 : (tok >= a.vocab ? a.vocab - 1 : tok);
    if (a.pos) {
      ps = a.positions[row];
      ps = ps < 0 ? 0 : (ps >= a.max_positions ? a.max_positions - 1 : ps);
    }
  }
#pragma unroll
  for (int k = 0; k < kMaxPieces; ++k) {
    const int pc = tid + k * THREADS;
    if (pc < pieces) {
      const int64_t at = row * a.width + pc * 8;
      float r[8];
      if (EMBED) {
        Vec8<T>::ld(a.embed, tok * a.width + pc * 8, v[k]);
#pragma unroll
        for (int i = 0; i < 8; ++i) v[k][i] *= a.embed_scale;
        if (a.pos) {
          Vec8<T>::ld(a.pos, ps * a.width + pc * 8, r);
#pragma unroll
          for (int i = 0; i < 8; ++i) v[k][i] += r[i];
        }
      } else {
        Vec8<F32>::ld(a.x, at, v[k]);
        if constexpr (NORMED > 0) {
#pragma unroll
          for (int b = 0; b < NB; ++b) {
            Vec8<F32>::ld(a.br[b].w, pc * 8, r);
#pragma unroll
            for (int i = 0; i < 8; ++i) v[k][i] += y[b][k][i] * ry[b] * r[i];
          }
        }
        for (int b = NORMED; b < a.n_br; ++b)
          for (int j = 0; j < a.br[b].n; ++j) {
            Vec8<T>::ld(a.br[b].y, j * a.y_plane + at, r);
#pragma unroll
            for (int i = 0; i < 8; ++i) v[k][i] += r[i];
          }
      }
      if (a.result) Vec8<F32>::st(a.result, at, v[k]);
      if (!EMBED && a.mix) {
        const float own = a.mix[a.n_hist];
#pragma unroll
        for (int i = 0; i < 8; ++i) v[k][i] *= own;
        int j = 0;
        for (; j + 4 <= a.n_hist; j += 4) {
          float h[4][8];
#pragma unroll
          for (int u = 0; u < 4; ++u) Vec8<F32>::ld(a.hist, (j + u) * a.hist_plane + at, h[u]);
#pragma unroll
          for (int u = 0; u < 4; ++u) {
            const float m = a.mix[j + u];
#pragma unroll
            for (int i = 0; i < 8; ++i) v[k][i] += m * h[u][i];
          }
        }
        for (; j < a.n_hist; ++j) {
          float h[8];
          Vec8<F32>::ld(a.hist, j * a.hist_plane + at, h);
          const float m = a.mix[j];
#pragma unroll
          for (int i = 0; i < 8; ++i) v[k][i] += m * h[i];
        }
      }
      if (a.shift) {
        Vec8<F32>::ld(a.shift, pc * 8, r);
#pragma unroll
        for (int i = 0; i < 8; ++i) v[k][i] += r[i];
      }
      if (a.x_out) Vec8<F32>::st(a.x_out, at, v[k]);
#pragma unroll
      for (int i = 0; i < 8; ++i) ss += v[k][i] * v[k][i];
    }
  }
  if (!a.w) return;
  if (a.b) {                               // no statistics: nothing to wait for
#pragma unroll
    for (int k = 0; k < kMaxPieces; ++k) {
      const int pc = tid + k * THREADS;
      if (pc < pieces) {
        float wv[8], bv[8];
        Vec8<F32>::ld(a.w, pc * 8, wv);
        Vec8<F32>::ld(a.b, pc * 8, bv);
#pragma unroll
        for (int i = 0; i < 8; ++i) v[k][i] = (tanh_of<T>(a.alpha * v[k][i]) * (a.offset + wv[i]) + bv[i]) * a.out_scale;
        Vec8<T>::st(a.out, row * a.width + pc * 8, v[k]);
      }
    }
    return;
  }
  ss = row_sum<kW>(ss, red, tid);
  const float rs = 1.f / sqrtf(ss / (float)a.norm_width + a.eps);
#pragma unroll
  for (int k = 0; k < kMaxPieces; ++k) {
    const int pc = tid + k * THREADS;
    if (pc < pieces) {
      float wv[8];
      Vec8<F32>::ld(a.w, pc * 8, wv);
#pragma unroll
      for (int i = 0; i < 8; ++i) v[k][i] = v[k][i] * rs * (a.offset + wv[i]) * a.out_scale;
      Vec8<T>::st(a.out, row * a.width + pc * 8, v[k]);
    }
  }
}

template <bool EMBED, int NORMED = 0>
int launch_rows(const RowArgs& a, int n, int dtype, hipStream_t st) {
  const bool small = a.width <= 512;
#define ZP_ROWS(T)                                                                             \
  do {                                                                                         \
    if (small) hipLaunchKernelGGL((row_kernel<T, 64, EMBED, NORMED>), dim3(n), dim3(64), 0, st, a);    \
    else hipLaunchKernelGGL((row_kernel<T, 256, EMBED, NORMED>), dim3(n), dim3(256), 0, st, a);        \
  } while (0)
  if (dtype == ZP_BF16) ZP_ROWS(BF16); else ZP_ROWS(F32);
#undef ZP_ROWS
  ZP_LAUNCH_CHECK();
  return ZP_OK;
}

// ------------------------------------------------------------------ activations
template <typename T>
__global__ __launch_bounds__(256) void relu_square_kernel(const void* in, void* out, int64_t pieces) {
  const int64_t id = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (id >= pieces) return;
  float z[8];
  Vec8<T>::ld(in, id * 8, z);
#pragma unroll
  for (int i = 0; i < 8; ++i) {
    const float r = fmaxf(z[i], 0.f);
    z[i] = r * r;
  }
  Vec8<T>::st(out, id * 8, z);
}

// z > 0: ap z^2 + z/2;  z <= 0: an (e^z - 1 - z) + z/2
template <typename T> __device__ __forceinline__ float expm1_minus(float z);
template <> __device__ __forceinline__ float expm1_minus<F32>(float z) { return expm1f(z) - z; }
template <> __device__ __forceinline__ float expm1_minus<BF16>(float z) {
  // near zero the Taylor series keeps the digits that the difference of near-equal terms loses
  const float series = z * z * (0.5f + z * (1.f / 6.f + z * (1.f / 24.f + z * (1.f / 120.f))));
  const float direct = __expf(z) - 1.f - z;
  return z > -0.125f ? series : direct;
}

template <typename T>
__global__ __launch_bounds__(256) void xielu_kernel(const void* in, void* out, int64_t pieces,
                                                    float ap, float an) {
  const int64_t id = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (id >= pieces) return;
  float z[8];
  Vec8<T>::ld(in, id * 8, z);
#pragma unroll
  for (int i = 0; i < 8; ++i) {
    const float pos = ap * z[i] * z[i];
    const float neg = an * expm1_minus<T>(fminf(z[i], 0.f));
    z[i] = (z[i] > 0.f ? pos : neg) + 0.5f * z[i];
  }
  Vec8<T>::st(out, id * 8, z);
}

// a N(z) + b N(z^2) + c N(z^3) + e, N dividing a row by its root mean square.  A workgroup per row, which
// stays in registers while its second, fourth and sixth powers are added up.
struct PowersArgs {
  const void* in;
  void* out;
  int width, norm_width;    // padded row length, and the length the means run over
  int64_t in_st, out_st;
  float a, b, c, e, eps;
};

template <typename T, int THREADS, int PIECES>
__global__ __launch_bounds__(THREADS) void normed_powers_kernel(PowersArgs a) {
  constexpr int kW = THREADS / 64;
  __shared__ float red[3][kW];
  const int tid = threadIdx.x;
  const int64_t row = blockIdx.x;
  const int pieces = a.width / 8;
  float z[PIECES][8], s[3] = {0.f, 0.f, 0.f};
#pragma unroll
  for (int k = 0; k < PIECES; ++k) {
    const int pc = tid + k * THREADS;
    if (pc < pieces) Vec8<T>::ld(a.in, row * a.in_st + pc * 8, z[k]);
    else {
#pragma unroll
      for (int i = 0; i < 8; ++i) z[k][i] = 0.f;
    }
  }
#pragma unroll
  for (int k = 0; k < PIECES; ++k)
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      const float q = z[k][i] * z[k][i];
      s[0] += q;
      s[1] = fmaf(q, q, s[1]);
      s[2] = fmaf(q * q, q, s[2]);
    }
#pragma unroll
  for (int j = 0; j < 3; ++j) {
    s[j] = wave_sum(s[j]);
    if (kW > 1 && (tid & 63) == 0) red[j][tid >> 6] = s[j];
  }
  if (kW > 1) {
    __syncthreads();
#pragma unroll
    for (int j = 0; j < 3; ++j) {
      s[j] = 0.f;
#pragma unroll
      for (int i = 0; i < kW; ++i) s[j] += red[j][i];
    }
  }
  const float inv = 1.f / (float)a.norm_width;
  const float f1 = a.a / sqrtf(s[0] * inv + a.eps), f2 = a.b / sqrtf(s[1] * inv + a.eps), f3 = a.c / sqrtf(s[2] * inv + a.eps);
#pragma unroll
  for (int k = 0; k < PIECES; ++k) {
    const int pc = tid + k * THREADS;
    if (pc < pieces) {
#pragma unroll
      for (int i = 0; i < 8; ++i) z[k][i] = fmaf(z[k][i], fmaf(z[k][i], fmaf(z[k][i], f3, f2), f1), a.e);
      Vec8<T>::st(a.out, row * a.out_st + pc * 8, z[k]);
    }
  }
}

template <typename T> void launch_powers(const PowersArgs& a, int n, hipStream_t st) {
  const int pieces = a.width / 8;
  if (pieces <= 64) hipLaunchKernelGGL((normed_powers_kernel<T, 64, 1>), dim3(n), dim3(64), 0, st, a);
  else if (pieces <= 256) hipLaunchKernelGGL((normed_powers_kernel<T, 256, 1>), dim3(n), dim3(256), 0, st, a);
  else if (pieces <= 1024) hipLaunchKernelGGL((normed_powers_kernel<T, 256, 4>), dim3(n), dim3(256), 0, st, a);
  else if (pieces <= 2048) hipLaunchKernelGGL((normed_powers_kernel<T, 512, 4>), dim3(n), dim3(512), 0, st, a);
  else if (pieces <= 3072) hipLaunchKernelGGL((normed_powers_kernel<T, 1024, 3>), dim3(n), dim3(1024), 0, st, a);
  else hipLaunchKernelGGL((normed_powers_kernel<T, 1024, 4>), dim3(n), dim3(1024), 0, st, a);
}

// ------------------------------------------------------------------ soft cap
// Logits leave in fp32: cap * tanh(z / cap).
template <typename T>
__global__ __launch_bounds__(256) void softcap_kernel(const void* in, float* out, int64_t count, float cap, float inv) {
  const int64_t i = ((int64_t)blockIdx.x * 256 + threadIdx.x) * 8;
  if (i >= count) return;
  if (i + 8 <= count) {
    float z[8];
    Vec8<T>::ld(in, i, z);
#pragma unroll
    for (int k = 0; k < 8; ++k) z[k] = cap * tanhf(z[k] * inv);
    Vec8<F32>::st(out, i, z);
  } else {
    for (int64_t k = i; k < count; ++k) out[k] = cap * tanhf(Elem<T>::ld(in, k) * inv);
  }
}

}  // namespace

#define ZP_ROW_WIDTH(name)                                                                      \
  if (width % 8 != 0 || width > 8 * 256 * kMaxPieces) {                                         \
    zp_set_error(name ": width %d unsupported (multiple of 8, <= %d)", width, 8 * 256 * kMaxPieces); \
    return ZP_EUNSUPPORTED;                                                                     \
  }

extern "C" int zp_embed_norm(const int64_t* tokens, const int32_t* positions, const void* embed,
                             const void* pos, const float* shift, float* result, float* x, const float* norm_weight,
                             const float* norm_bias, void* out, int32_t n, int32_t width, int32_t norm_width,
                             int64_t vocab, int64_t max_positions, float embed_scale, float eps,
                             float weight_offset, float norm_alpha, int32_t dtype, void* stream) {
  ZP_REQUIRE(n >= 0 && width > 0 && norm_width > 0 && norm_width <= width && vocab > 0,
             "embed_norm: bad dims");
  ZP_MODEL_DTYPE("embed_norm");
  ZP_ROW_WIDTH("embed_norm");
  if (n == 0) return ZP_OK;
  ZP_REQUIRE(tokens && embed && x && (!pos || (positions && max_positions > 0)) &&
                 (!norm_weight || out), "embed_norm: null pointer");
  ZP_REQUIRE(aligned16(embed) && aligned16(pos) && aligned16(x) && aligned16(norm_weight) && aligned16(norm_bias) && aligned16(out) &&
                 aligned16(shift) && aligned16(result),
             "embed_norm: tensors must be 16-byte aligned");
  RowArgs a = {};
  a.tokens = tokens; a.positions = positions; a.embed = embed; a.pos = pos; a.vocab = vocab;
  a.max_positions = max_positions; a.shift = shift; a.result = result; a.x_out = x; a.w = norm_weight; a.out = out; a.width = width;
  a.norm_width = norm_width; a.eps = eps; a.offset = weight_offset; a.out_scale = 1.f;
  a.embed_scale = embed_scale; a.b = norm_bias; a.alpha = norm_alpha;
  return launch_rows<true>(a, n, dtype, (hipStream_t)stream);
}

extern "C" int zp_residual_norm(const float* x, const zp_branch* branches, int32_t n_branches,
                                const float* hist, int64_t hist_plane, const float* mix, int32_t n_hist,
                                const float* shift, float* result, float* x_out, const float* norm_weight,
                                const float* norm_bias, void* out, int32_t n, int32_t width, int32_t norm_width, float eps,
                                float weight_offset, float norm_alpha, float out_scale, int32_t dtype, void* stream) {
  ZP_REQUIRE(n >= 0 && width > 0 && norm_width > 0 && norm_width <= width && n_hist >= 0 && branches && n_branches >= 1 &&
                 n_branches <= kMaxBranches, "residual_norm: bad dims");
  ZP_MODEL_DTYPE("residual_norm");
  ZP_ROW_WIDTH("residual_norm");
  if (n == 0) return ZP_OK;
  RowArgs a = {};
  int normed = 0;
  for (int pass = 0; pass < 2; ++pass)          // those with a norm first
    for (int i = 0; i < n_branches; ++i) {
      const zp_branch& b = branches[i];
      ZP_REQUIRE(b.y && b.planes >= 1 && aligned16(b.y) && aligned16(b.weight), "residual_norm: a branch is missing or unaligned");
      if ((b.weight != nullptr) != (pass == 0)) continue;
      a.br[a.n_br++] = Branch{b.y, b.weight, b.planes};
      normed += pass == 0;
    }
  ZP_REQUIRE(normed <= kMaxNormed, "residual_norm: at most %d branches are normed", kMaxNormed);
  ZP_REQUIRE(x && (!norm_weight || out), "residual_norm: null pointer");
  ZP_REQUIRE(n_hist == 0 || (hist && mix && hist_plane >= (int64_t)n * width),
             "residual_norm: a depth average needs its weights and planes of n rows");
  ZP_REQUIRE(aligned16(x) && aligned16(hist) && hist_plane % 4 == 0 && aligned16(shift) && aligned16(result) &&
                 aligned16(x_out) && aligned16(norm_weight) && aligned16(norm_bias) && aligned16(out),
             "residual_norm: tensors must be 16-byte aligned");
  a.x = x; a.y_plane = (int64_t)n * width; a.hist = hist; a.hist_plane = hist_plane; a.mix = mix; a.n_hist = n_hist;
  a.shift = shift; a.result = result; a.x_out = x_out; a.w = norm_weight; a.out = out; a.width = width;
  a.norm_width = norm_width; a.eps = eps; a.offset = weight_offset; a.out_scale = out_scale;
  a.b = norm_bias; a.alpha = norm_alpha;
  hipStream_t st = (hipStream_t)stream;
  switch (normed) {
    case 0: return launch_rows<false>(a, n, dtype, st);
    case 1: return launch_rows<false, 1>(a, n, dtype, st);
    default: return launch_rows<false, 2>(a, n, dtype, st);
  }
}

extern "C" int zp_xielu(const void* in, void* out, int64_t count, float alpha_p, float alpha_n,
                        int32_t dtype, void* stream) {
  ZP_REQUIRE(count >= 0 && count % 8 == 0, "xielu: element count must be a multiple of 8");
  ZP_MODEL_DTYPE("xielu");
  if (count == 0) return ZP_OK;
  ZP_REQUIRE(in && out && aligned16(in) && aligned16(out), "xielu: null or unaligned pointer");
  const int64_t pieces = count / 8;
  const unsigned grid = (unsigned)((pieces + 255) / 256);
  hipStream_t st = (hipStream_t)stream;
  if (dtype == ZP_BF16)
    hipLaunchKernelGGL((xielu_kernel<BF16>), dim3(grid), dim3(256), 0, st, in, out, pieces, alpha_p, alpha_n);
  else
    hipLaunchKernelGGL((xielu_kernel<F32>), dim3(grid), dim3(256), 0, st, in, out, pieces, alpha_p, alpha_n);
  ZP_LAUNCH_CHECK();
  return ZP_OK;
}

extern "C" int zp_relu_square(const void* in, void* out, int64_t count, int32_t dtype, void* stream) {
  ZP_REQUIRE(count >= 0 && count % 8 == 0, "relu_square: element count must be a multiple of 8");
  ZP_MODEL_DTYPE("relu_square");
  if (count == 0) return ZP_OK;
  ZP_REQUIRE(in && out && aligned16(in) && aligned16(out), "relu_square: null or unaligned pointer");
  const int64_t pieces = count / 8;
  const unsigned grid = (unsigned)((pieces + 255) / 256);
  hipStream_t st = (hipStream_t)stream;
  if (dtype == ZP_BF16) hipLaunchKernelGGL((relu_square_kernel<BF16>), dim3(grid), dim3(256), 0, st, in, out, pieces);
  else hipLaunchKernelGGL((relu_square_kernel<F32>), dim3(grid), dim3(256), 0, st, in, out, pieces);
  ZP_LAUNCH_CHECK();
  return ZP_OK;
}

extern "C" int zp_normed_powers(const void* in, void* out, int32_t n, int32_t width, int32_t norm_width,
                                int64_t in_stride, int64_t out_stride, float a, float b, float c, float e, float eps,
                                int32_t dtype, void* stream) {
  ZP_REQUIRE(n >= 0 && width > 0 && norm_width > 0 && norm_width <= width && in_stride >= width && out_stride >= width,
             "normed_powers: bad dims");
  ZP_MODEL_DTYPE("normed_powers");
  if (width % 8 != 0 || width > 32768 || in_stride % 8 != 0 || out_stride % 8 != 0) {
    zp_set_error("normed_powers: width %d unsupported (a multiple of 8, <= 32768)", width);
    return ZP_EUNSUPPORTED;
  }
  if (n == 0) return ZP_OK;
  ZP_REQUIRE(in && out && aligned16(in) && aligned16(out), "normed_powers: null or unaligned pointer");
  const PowersArgs args = {in, out, width, norm_width, in_stride, out_stride, a, b, c, e, eps};
  if (dtype == ZP_BF16) launch_powers<BF16>(args, n, (hipStream_t)stream);
  else launch_powers<F32>(args, n, (hipStream_t)stream);
  ZP_LAUNCH_CHECK();
  return ZP_OK;
}

extern "C" int zp_softcap(const void* in, float* out, int64_t count, float cap, int32_t dtype, void* stream) {
  ZP_REQUIRE(count >= 0 && cap > 0.f, "softcap: bad arguments");
  ZP_MODEL_DTYPE("softcap");
  if (count == 0) return ZP_OK;
  ZP_REQUIRE(in && out && aligned16(in) && aligned16(out), "softcap: null or unaligned pointer");
  const unsigned grid = (unsigned)((count + 2047) / 2048);
  hipStream_t st = (hipStream_t)stream;
  if (dtype == ZP_BF16) hipLaunchKernelGGL((softcap_kernel<BF16>), dim3(grid), dim3(256), 0, st, in, out, count, cap, 1.f / cap);
  else hipLaunchKernelGGL((softcap_kernel<F32>), dim3(grid), dim3(256), 0, st, in, out, count, cap, 1.f / cap);
  ZP_LAUNCH_CHECK();
  return ZP_OK;
}
