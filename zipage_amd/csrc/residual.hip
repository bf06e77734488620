// Row kernels of decoders that keep their residual stream in fp32 whatever the dtype of their
// matrix products: token + learned-position embedding, residual add (of a branch output as it is or
// normed), depth average over all earlier layer results, RMS norm or tanh norm, the xIELU and squared
// relu activations, and the soft cap of logits.  Each is one pass over its rows (HBM- or
// launch-bound): the stream is read once, and what the next matrix product needs leaves the same
// launch in that product's dtype.
#include "models.h"
#include <math.h>

namespace {

constexpr int kMaxPieces = 4;   // 8-element pieces per thread: rows up to 8 * 4 * 256 elements

struct RowArgs {
  // source: an embedding (tokens, positions) or the stream x plus a branch output y
  const int64_t* tokens;
  const int32_t* positions;
  const void* embed;      // (vocab, width) T
  const void* pos;        // (max_positions, width) T or null
  int64_t vocab, max_positions;
  const float* x;         // (n, width) fp32
  const void* y;          // n_y planes of (n, width) T
  int64_t y_plane;
  int n_y;
  const float* yw;        // (width,) weight of an RMS norm on y before the add, or null
  float embed_scale;
  // depth average: result_new = sum_j mix[j] * hist[j] + mix[n_hist] * (x + y)
  const float* hist;      // n_hist planes of (n, width) fp32
  int64_t hist_plane;     // elements between planes
  const float* mix;       // n_hist + 1 weights, or null: the sum itself goes on
  int n_hist;
  float* result;          // receives x + y before the average, or null
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

template <typename T, int THREADS, bool EMBED, bool BRANCH>
__global__ __launch_bounds__(THREADS) void row_kernel(RowArgs a) {
  constexpr int kW = THREADS / 64;
  __shared__ float red[kW], red_y[kW];
  const int tid = threadIdx.x;
  const int64_t row = blockIdx.x;
  const int pieces = a.width / 8;
  float v[kMaxPieces][8];
  float ss = 0.f;
  float y[BRANCH ? kMaxPieces : 1][8];     // the normed branch: its sum first, the stream joins later
  float ry = 0.f;
  if constexpr (BRANCH) {
#pragma unroll
    for (int k = 0; k < kMaxPieces; ++k) {
      const int pc = tid + k * THREADS;
      if (pc < pieces) {
        const int64_t at = row * a.width + pc * 8;
        Vec8<T>::ld(a.y, at, y[k]);
        int j = 1;
        for (; j + 4 <= a.n_y; j += 4) {
          float r[4][8];
#pragma unroll
          for (int u = 0; u < 4; ++u) Vec8<T>::ld(a.y, (j + u) * a.y_plane + at, r[u]);
#pragma unroll
          for (int u = 0; u < 4; ++u)
#pragma unroll
            for (int i = 0; i < 8; ++i) y[k][i] += r[u][i];
        }
        for (; j < a.n_y; ++j) {
          float r[8];
          Vec8<T>::ld(a.y, j * a.y_plane + at, r);
#pragma unroll
          for (int i = 0; i < 8; ++i) y[k][i] += r[i];
        }
#pragma unroll
        for (int i = 0; i < 8; ++i) ry += y[k][i] * y[k][i];
      }
    }
    ry = 1.f / sqrtf(row_sum<kW>(ry, red_y, tid) / (float)a.norm_width + a.eps);
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
        if constexpr (BRANCH) {
          Vec8<F32>::ld(a.yw, pc * 8, r);
#pragma unroll
          for (int i = 0; i < 8; ++i) v[k][i] += y[k][i] * ry * r[i];
        } else for (int j = 0; j < a.n_y; ++j) {
          Vec8<T>::ld(a.y, j * a.y_plane + at, r);
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

template <bool EMBED, bool BRANCH = false>
int launch_rows(const RowArgs& a, int n, int dtype, hipStream_t st) {
  const bool small = a.width <= 512;
#define ZP_ROWS(T)                                                                             \
  do {                                                                                         \
    if (small) hipLaunchKernelGGL((row_kernel<T, 64, EMBED, BRANCH>), dim3(n), dim3(64), 0, st, a);    \
    else hipLaunchKernelGGL((row_kernel<T, 256, EMBED, BRANCH>), dim3(n), dim3(256), 0, st, a);        \
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
                             const void* pos, float* x, const float* norm_weight, const float* norm_bias,
                             void* out, int32_t n, int32_t width, int32_t norm_width, int64_t vocab,
                             int64_t max_positions, float embed_scale, float eps, float weight_offset,
                             float norm_alpha, int32_t dtype, void* stream) {
  ZP_REQUIRE(n >= 0 && width > 0 && norm_width > 0 && norm_width <= width && vocab > 0,
             "embed_norm: bad dims");
  ZP_MODEL_DTYPE("embed_norm");
  ZP_ROW_WIDTH("embed_norm");
  if (n == 0) return ZP_OK;
  ZP_REQUIRE(tokens && embed && x && (!pos || (positions && max_positions > 0)) &&
                 (!norm_weight || out), "embed_norm: null pointer");
  ZP_REQUIRE(aligned16(embed) && aligned16(pos) && aligned16(x) && aligned16(norm_weight) && aligned16(norm_bias) && aligned16(out),
             "embed_norm: tensors must be 16-byte aligned");
  RowArgs a = {};
  a.tokens = tokens; a.positions = positions; a.embed = embed; a.pos = pos; a.vocab = vocab;
  a.max_positions = max_positions; a.x_out = x; a.w = norm_weight; a.out = out; a.width = width;
  a.norm_width = norm_width; a.eps = eps; a.offset = weight_offset; a.out_scale = 1.f;
  a.embed_scale = embed_scale; a.b = norm_bias; a.alpha = norm_alpha;
  return launch_rows<true>(a, n, dtype, (hipStream_t)stream);
}

extern "C" int zp_residual_norm(const float* x, const void* y, int32_t n_y, const float* y_weight,
                                const float* hist, int64_t hist_plane, const float* mix, int32_t n_hist,
                                float* result, float* x_out, const float* norm_weight, const float* norm_bias, void* out,
                                int32_t n, int32_t width, int32_t norm_width, float eps,
                                float weight_offset, float norm_alpha, float out_scale, int32_t dtype, void* stream) {
  ZP_REQUIRE(n >= 0 && width > 0 && norm_width > 0 && norm_width <= width && n_hist >= 0 && n_y >= 1,
             "residual_norm: bad dims");
  ZP_MODEL_DTYPE("residual_norm");
  ZP_ROW_WIDTH("residual_norm");
  if (n == 0) return ZP_OK;
  ZP_REQUIRE(x && y && (!norm_weight || out), "residual_norm: null pointer");
  ZP_REQUIRE(n_hist == 0 || (hist && mix && hist_plane >= (int64_t)n * width),
             "residual_norm: a depth average needs its weights and planes of n rows");
  ZP_REQUIRE(aligned16(x) && aligned16(y) && aligned16(y_weight) && aligned16(hist) && hist_plane % 4 == 0 && aligned16(result) &&
                 aligned16(x_out) && aligned16(norm_weight) && aligned16(norm_bias) && aligned16(out),
             "residual_norm: tensors must be 16-byte aligned");
  RowArgs a = {};
  a.x = x; a.y = y; a.n_y = n_y; a.y_plane = (int64_t)n * width; a.hist = hist; a.hist_plane = hist_plane; a.mix = mix; a.n_hist = n_hist;
  a.result = result; a.x_out = x_out; a.w = norm_weight; a.out = out; a.width = width;
  a.norm_width = norm_width; a.eps = eps; a.offset = weight_offset; a.out_scale = out_scale;
  a.yw = y_weight; a.b = norm_bias; a.alpha = norm_alpha;
  if (y_weight) return launch_rows<false, true>(a, n, dtype, (hipStream_t)stream);
  return launch_rows<false>(a, n, dtype, (hipStream_t)stream);
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
