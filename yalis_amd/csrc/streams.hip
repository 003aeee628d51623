// A residual stream kept as several copies x_1 .. x_S [tokens][S][width], float32:
//
//   y   = dense[n, :] + weight * sum_k row_weights[n, k] rows[n top + k, :]     (a branch's output, any of its parts)
//   x_t <- sum_s mix[s, t] x_s + out[t] y                                       (all t from the old x_s)
//   h   = norm(sum_t read[t] x_t)                                               (what the next branch reads)
//
// in one pass over a token's copies (yk_streams_norm): a thread holds four neighbouring elements of every copy, so the old
// copies are read once, the new ones written once, and the sum that is normed never leaves the registers.  The branch may be
// a tensor, a product's unreduced K slices (float32, summed in order and rounded as the product's output would have been),
// and / or the uncombined rows of a mixture's experts.  `rows` picks token rows and leaves the copies as they are: the final
// norm on the rows whose logits are wanted (read null: the plain sum).
//
// Beside it yk_embed_norm, with which such a stream starts: a token's row of the embedding table through an RMS norm with a
// weight, written once per copy.
#include <algorithm>

#include "common.h"

constexpr int kMaxStreams = 16;

struct StreamsArgs {
  int n_splits;
  size_t split_stride;
  int round_sum;
  const float* expert_rows;
  int top;
  float expert_weight;
  const float* row_weights;
  const float *mix, *out, *read;
  const int32_t* rows;
  float eps;
  int unit_offset, width, streams;
};

template <typename T>
__device__ __forceinline__ float4 st_load4(const T* p);
template <>
__device__ __forceinline__ float4 st_load4<float>(const float* p) {
  return *reinterpret_cast<const float4*>(p);
}
template <>
__device__ __forceinline__ float4 st_load4<bf16_t>(const bf16_t* p) {
  const uint2 w = *reinterpret_cast<const uint2*>(p);
  return make_float4(__uint_as_float(w.x << 16), __uint_as_float(w.x & 0xffff0000u), __uint_as_float(w.y << 16),
                     __uint_as_float(w.y & 0xffff0000u));
}
template <typename T>
__device__ __forceinline__ void st_store4(T* p, float4 v);
template <>
__device__ __forceinline__ void st_store4<float>(float* p, float4 v) {
  *reinterpret_cast<float4*>(p) = v;
}
template <>
__device__ __forceinline__ void st_store4<bf16_t>(bf16_t* p, float4 v) {
  *reinterpret_cast<uint2*>(p) = make_uint2(pack_bf16x2(v.x, v.y), pack_bf16x2(v.z, v.w));
}
__device__ __forceinline__ void st_fma4(float4& a, float m, const float4& v) {
  a.x = fmaf(m, v.x, a.x);
  a.y = fmaf(m, v.y, a.y);
  a.z = fmaf(m, v.z, a.z);
  a.w = fmaf(m, v.w, a.w);
}

// P pieces of four elements a thread (width <= 4 P blockDim), up to SMAX copies
template <int SMAX, int P, typename TS, typename TW, typename TO>
__global__ __launch_bounds__(1024) void streams_norm_vec_kernel(float* __restrict__ x, const TS* __restrict__ y, const TW* __restrict__ weight,
                                                                TO* __restrict__ h, StreamsArgs g) {
  __shared__ float scratch[17];
  const size_t n = blockIdx.x, r = g.rows != nullptr ? static_cast<size_t>(g.rows[n]) : n;
  const int S = g.streams, width = g.width;
  float* xr = x + r * S * width;
  float4 u[P], w[P];
  float ss = 0.f;
#pragma unroll
  for (int p = 0; p < P; ++p) {
    const int c = 4 * (threadIdx.x + p * blockDim.x);
    u[p] = w[p] = make_float4(0.f, 0.f, 0.f, 0.f);
    if (c < width) {
      float4 xs[SMAX];
#pragma unroll
      for (int s = 0; s < SMAX; ++s)
        if (s < S) xs[s] = *reinterpret_cast<const float4*>(xr + static_cast<size_t>(s) * width + c);
      w[p] = st_load4<TW>(weight + c);
      if (g.mix == nullptr) {
#pragma unroll
        for (int s = 0; s < SMAX; ++s)
          if (s < S) st_fma4(u[p], g.read != nullptr ? g.read[s] : 1.f, xs[s]);
      } else {
        float4 b = make_float4(0.f, 0.f, 0.f, 0.f);
        if (y != nullptr) {
          for (int s0 = 0; s0 < g.n_splits; s0 += 8) {
            float4 t[8];
#pragma unroll
            for (int j = 0; j < 8; ++j)
              t[j] = st_load4<TS>(y + static_cast<size_t>(min(s0 + j, g.n_splits - 1)) * g.split_stride + r * width + c);
#pragma unroll
            for (int j = 0; j < 8; ++j)
              if (s0 + j < g.n_splits) b.x += t[j].x, b.y += t[j].y, b.z += t[j].z, b.w += t[j].w;
          }
          b = make_float4(as_output(b.x, g.round_sum), as_output(b.y, g.round_sum), as_output(b.z, g.round_sum), as_output(b.w, g.round_sum));
        }
        if (g.expert_rows != nullptr) {
          float4 e = make_float4(0.f, 0.f, 0.f, 0.f);
          const float* er = g.expert_rows + r * g.top * width + c;
          for (int k0 = 0; k0 < g.top; k0 += 4) {
            float4 t[4];
            float m[4];
#pragma unroll
            for (int j = 0; j < 4; ++j) {
              const int k = min(k0 + j, g.top - 1);
              t[j] = *reinterpret_cast<const float4*>(er + static_cast<size_t>(k) * width);
              m[j] = g.row_weights != nullptr ? g.row_weights[r * g.top + k] : 1.f;
            }
#pragma unroll
            for (int j = 0; j < 4; ++j)
              if (k0 + j < g.top) st_fma4(e, m[j], t[j]);
          }
          st_fma4(b, g.expert_weight, e);
        }
#pragma unroll
        for (int t = 0; t < SMAX; ++t)
          if (t < S) {
            const float o = g.out[t];
            float4 v = make_float4(o * b.x, o * b.y, o * b.z, o * b.w);
#pragma unroll
            for (int s = 0; s < SMAX; ++s)
              if (s < S) st_fma4(v, g.mix[s * S + t], xs[s]);
            if (g.rows == nullptr) *reinterpret_cast<float4*>(xr + static_cast<size_t>(t) * width + c) = v;
            st_fma4(u[p], g.read != nullptr ? g.read[t] : 1.f, v);
          }
      }
      ss = fmaf(u[p].x, u[p].x, fmaf(u[p].y, u[p].y, fmaf(u[p].z, u[p].z, fmaf(u[p].w, u[p].w, ss))));
    }
  }
  const float inv = 1.f / sqrtf(block_sum(ss, scratch) / static_cast<float>(width) + g.eps);
  const float one = g.unit_offset ? 1.f : 0.f;
#pragma unroll
  for (int p = 0; p < P; ++p) {
    const int c = 4 * (threadIdx.x + p * blockDim.x);
    if (c < width)
      st_store4<TO>(h + n * width + c, make_float4(u[p].x * inv * (w[p].x + one), u[p].y * inv * (w[p].y + one), u[p].z * inv * (w[p].z + one),
                                                   u[p].w * inv * (w[p].w + one)));
  }
}

// any width and alignment: an element of every copy a thread at a time, the sum parked in LDS
template <typename TS, typename TW, typename TO>
__global__ __launch_bounds__(256) void streams_norm_kernel(float* __restrict__ x, const TS* __restrict__ y, const TW* __restrict__ weight,
                                                           TO* __restrict__ h, StreamsArgs g) {
  extern __shared__ float row[];  // [width], then 17 floats of scratch
  const size_t n = blockIdx.x, r = g.rows != nullptr ? static_cast<size_t>(g.rows[n]) : n;
  const int S = g.streams, width = g.width;
  float* scratch = row + width;
  float* xr = x + r * S * width;
  float ss = 0.f;
  for (int c = threadIdx.x; c < width; c += blockDim.x) {
    float xs[kMaxStreams];
#pragma unroll
    for (int s = 0; s < kMaxStreams; ++s) xs[s] = s < S ? xr[static_cast<size_t>(s) * width + c] : 0.f;
    float u = 0.f;
    if (g.mix == nullptr) {
#pragma unroll
      for (int s = 0; s < kMaxStreams; ++s)
        if (s < S) u = fmaf(g.read != nullptr ? g.read[s] : 1.f, xs[s], u);
    } else {
      float b = 0.f;
      if (y != nullptr) {
        for (int s = 0; s < g.n_splits; ++s) b += to_f32<TS>(y[s * g.split_stride + r * width + c]);
        b = as_output(b, g.round_sum);
      }
      if (g.expert_rows != nullptr) {
        float e = 0.f;
        for (int k = 0; k < g.top; ++k)
          e = fmaf(g.row_weights != nullptr ? g.row_weights[r * g.top + k] : 1.f, g.expert_rows[(r * g.top + k) * width + c], e);
        b = fmaf(g.expert_weight, e, b);
      }
      for (int t = 0; t < S; ++t) {
        float v = g.out[t] * b;
#pragma unroll
        for (int s = 0; s < kMaxStreams; ++s)
          if (s < S) v = fmaf(g.mix[s * S + t], xs[s], v);
        if (g.rows == nullptr) xr[static_cast<size_t>(t) * width + c] = v;
        u = fmaf(g.read != nullptr ? g.read[t] : 1.f, v, u);
      }
    }
    row[c] = u;
    ss = fmaf(u, u, ss);
  }
  const float inv = 1.f / sqrtf(block_sum(ss, scratch) / static_cast<float>(width) + g.eps);
  for (int c = threadIdx.x; c < width; c += blockDim.x)
    h[n * width + c] = from_f32<TO>(row[c] * inv * (to_f32<TW>(weight[c]) + (g.unit_offset ? 1.f : 0.f)));
}

// x_rows: tokens of x (and of every slice of y: the stride between slices); n_rows: rows of h.  mix null: nothing is pending.
extern "C" int yk_streams_norm(float* x, int x_rows, int streams, int width, const void* y, int y_dtype, int n_splits, int round_sum,
                               const float* expert_rows, int top, float expert_weight, const float* row_weights, const float* mix,
                               const float* out, const float* read, const int32_t* rows, const void* weight, int w_dtype, float eps,
                               int unit_offset, void* h, int h_dtype, int n_rows, hipStream_t stream) {
  YK_REQUIRE(x != nullptr && x_rows >= 0 && n_rows >= 0 && width > 0 && streams >= 1 && streams <= kMaxStreams, "streams_norm: bad sizes (up to 16 copies)");
  YK_REQUIRE(rows != nullptr || n_rows == x_rows, "streams_norm: a row of the result per token, or rows that are picked");
  YK_REQUIRE((mix != nullptr) == (out != nullptr) && (mix != nullptr || (y == nullptr && expert_rows == nullptr)),
             "streams_norm: a branch joins through both of its tables");
  YK_REQUIRE(n_splits >= 1 && (n_splits == 1 || y_dtype == YK_F32), "streams_norm: unreduced slices must be float32");
  YK_REQUIRE(expert_rows == nullptr || top >= 1, "streams_norm: bad expert rows");
  if (n_rows == 0) return 0;
  const StreamsArgs g{n_splits, static_cast<size_t>(x_rows) * width, round_sum, expert_rows, top, expert_weight, row_weights, mix, out, read,
                      rows, eps, unit_offset, width, streams};
  auto al = [](const void* p) { return reinterpret_cast<uintptr_t>(p) % 16 == 0; };
  const bool vec = width % 4 == 0 && width <= 16384 && al(x) && al(y) && al(expert_rows) && al(weight) && al(h);
  const int threads = std::min(1024, (width / 4 + 63) / 64 * 64);
  const size_t lds = (static_cast<size_t>(width) + 17) * sizeof(float);
  YK_REQUIRE(vec || width <= 15 * 1024, "streams_norm: rows of more than 15,360 elements do not fit the row buffer");
#define YK_VEC(SM, PP, TS, TW, TO)                                                                                                \
  streams_norm_vec_kernel<SM, PP, TS, TW, TO><<<n_rows, threads, 0, stream>>>(x, static_cast<const TS*>(y), static_cast<const TW*>(weight), \
                                                                             static_cast<TO*>(h), g)
#define YK_CASE(SD, TS, WD, TW, OD, TO)                                                                                           \
  if ((y == nullptr || y_dtype == SD) && w_dtype == WD && h_dtype == OD) {                                                        \
    if (vec && width <= 4096) {                                                                                                   \
      if (streams <= 4) YK_VEC(4, 1, TS, TW, TO);                                                                                 \
      else if (streams <= 8) YK_VEC(8, 1, TS, TW, TO);                                                                            \
      else YK_VEC(16, 1, TS, TW, TO);                                                                                             \
    } else if (vec) {                                                                                                             \
      if (streams <= 4) YK_VEC(4, 4, TS, TW, TO);                                                                                 \
      else YK_VEC(16, 4, TS, TW, TO);                                                                                             \
    } else {                                                                                                                      \
      streams_norm_kernel<TS, TW, TO><<<n_rows, 256, lds, stream>>>(x, static_cast<const TS*>(y), static_cast<const TW*>(weight), \
                                                                    static_cast<TO*>(h), g);                                      \
    }                                                                                                                             \
    return yk_check_launch("streams_norm");                                                                                       \
  }
  YK_CASE(YK_F32, float, YK_F32, float, YK_F32, float)
  YK_CASE(YK_F32, float, YK_BF16, bf16_t, YK_BF16, bf16_t)
  YK_CASE(YK_BF16, bf16_t, YK_BF16, bf16_t, YK_BF16, bf16_t)
  YK_CASE(YK_F32, float, YK_F32, float, YK_BF16, bf16_t)
  YK_CASE(YK_BF16, bf16_t, YK_F32, float, YK_BF16, bf16_t)
#undef YK_CASE
#undef YK_VEC
  return yk_fail("streams_norm: unsupported dtype combination");
}

// ---------------------------------------------------------------------------- the stream's start
// out[n, s, :] = table[ids[n]] / sqrt(mean(table[ids[n]]^2) + eps) * weight for every copy s.  A workgroup a token.
template <typename T, bool VEC>
__global__ __launch_bounds__(256) void embed_norm_kernel(const int32_t* __restrict__ ids, const T* __restrict__ table, int vocab,
                                                         const T* __restrict__ weight, float eps, float* __restrict__ out, int width,
                                                         int copies) {
  __shared__ float scratch[17];
  const size_t n = blockIdx.x;
  const int id = min(max(ids[n], 0), vocab - 1);  // (ids are checked on the host; clamped so that a bad id cannot read out of bounds)
  const T* src = table + static_cast<size_t>(id) * width;
  float* dst = out + n * copies * width;
  float ss = 0.f;
  if constexpr (VEC) {
    for (int c = 4 * threadIdx.x; c < width; c += 4 * blockDim.x) {
      const float4 v = st_load4<T>(src + c);
      ss = fmaf(v.x, v.x, fmaf(v.y, v.y, fmaf(v.z, v.z, fmaf(v.w, v.w, ss))));
    }
  } else {
    for (int c = threadIdx.x; c < width; c += blockDim.x) ss = fmaf(to_f32<T>(src[c]), to_f32<T>(src[c]), ss);
  }
  const float inv = 1.f / sqrtf(block_sum(ss, scratch) / static_cast<float>(width) + eps);
  if constexpr (VEC) {
    for (int c = 4 * threadIdx.x; c < width; c += 4 * blockDim.x) {
      const float4 v = st_load4<T>(src + c), w = st_load4<T>(weight + c);
      const float4 o = make_float4(v.x * inv * w.x, v.y * inv * w.y, v.z * inv * w.z, v.w * inv * w.w);
      for (int s = 0; s < copies; ++s) *reinterpret_cast<float4*>(dst + static_cast<size_t>(s) * width + c) = o;
    }
  } else {
    for (int c = threadIdx.x; c < width; c += blockDim.x) {
      const float o = to_f32<T>(src[c]) * inv * to_f32<T>(weight[c]);
      for (int s = 0; s < copies; ++s) dst[static_cast<size_t>(s) * width + c] = o;
    }
  }
}

extern "C" int yk_embed_norm(const int32_t* ids, const void* table, int dtype, int vocab, const void* weight, float eps, float* out,
                             int n_tokens, int width, int copies, hipStream_t stream) {
  YK_REQUIRE(n_tokens >= 0 && width > 0 && vocab > 0 && copies >= 1, "embed_norm: bad sizes");
  if (n_tokens == 0) return 0;
  auto al = [](const void* p) { return reinterpret_cast<uintptr_t>(p) % 16 == 0; };
  const bool vec = width % 4 == 0 && al(table) && al(weight) && al(out);
#define YK_CASE(D, T, V)                                                                                                            \
  if (dtype == D && vec == V) {                                                                                                     \
    embed_norm_kernel<T, V><<<n_tokens, 256, 0, stream>>>(ids, static_cast<const T*>(table), vocab, static_cast<const T*>(weight), eps, out, \
                                                          width, copies);                                                           \
    return yk_check_launch("embed_norm");                                                                                           \
  }
  YK_CASE(YK_F32, float, true)
  YK_CASE(YK_F32, float, false)
  YK_CASE(YK_BF16, bf16_t, true)
  YK_CASE(YK_BF16, bf16_t, false)
#undef YK_CASE
  return yk_fail("embed_norm: unsupported table dtype");
}
