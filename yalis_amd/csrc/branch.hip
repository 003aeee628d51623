// A branch's output joins the residual stream through a norm of its own:
//   residual[n, :] += branch[n, :] / sqrt(mean(branch[n, :]^2) + eps) * w'      (w' = w or 1 + w)
// and, where the engine's activations are narrower than the float32 residual, the new residual
// rounded to the activation dtype is written beside it: the next branch reads the stream itself,
// not a normed copy, so this is the only pass over the row between two branches.
//
// The branch may come as
//   * a tensor [rows, width] in the activation dtype or float32,
//   * the unreduced K slices of a product (float32 [slices, rows, width]; summed in the order of
//     the slices and, with round_sum, rounded as the product's own output would have been),
//   * and / or the rows of a mixture of experts before they are combined: float32
//     [rows * top, width], of which row n takes pair_weight * (the sum of its `top` rows, in
//     order).
// Everything is float32 arithmetic; one workgroup a row, the row parked in LDS between the
// sum of squares and the update.
//
// Beside it: the other arrangement, the stream itself normed after a branch has joined it (yk_sum_norm).
#include <algorithm>

#include "common.h"

// Four consecutive elements of a row of T as floats (16-byte aligned rows of a multiple of four).
template <typename T>
__device__ __forceinline__ float4 na_load4(const T* p);
template <>
__device__ __forceinline__ float4 na_load4<float>(const float* p) {
  return *reinterpret_cast<const float4*>(p);
}
template <>
__device__ __forceinline__ float4 na_load4<bf16_t>(const bf16_t* p) {
  const uint2 w = *reinterpret_cast<const uint2*>(p);
  return make_float4(__uint_as_float(w.x << 16), __uint_as_float(w.x & 0xffff0000u), __uint_as_float(w.y << 16),
                     __uint_as_float(w.y & 0xffff0000u));
}

// VEC: four columns a thread with 16-byte accesses, and the slices (or a token's expert rows) of a
// column asked for eight at a time before any is added: with one element a thread and one load
// behind the other, eight rows of 2,048 took 17 us of waiting.  The sums keep the order of the slices.
template <typename TS, typename TW, typename TO, bool VEC>
__global__ __launch_bounds__(256) void norm_add_kernel(
    float* __restrict__ residual, const TS* __restrict__ src, int n_splits, size_t split_stride, int round_sum,
    const float* __restrict__ pairs, int top, float pair_weight, const TW* __restrict__ w, int unit_offset,
    float eps, TO* __restrict__ out, int width) {
  extern __shared__ float row[];  // [width], then 17 floats of scratch
  float* scratch = row + width;
  const size_t n = blockIdx.x;
  float ss = 0.f;
  if (VEC) {
    for (int c = 4 * threadIdx.x; c < width; c += 4 * blockDim.x) {
      float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
      if (src != nullptr) {
        for (int s0 = 0; s0 < n_splits; s0 += 8) {
          float4 t[8];
#pragma unroll
          for (int j = 0; j < 8; ++j)
            if (s0 + j < n_splits) t[j] = na_load4<TS>(src + (s0 + j) * split_stride + n * width + c);
#pragma unroll
          for (int j = 0; j < 8; ++j)
            if (s0 + j < n_splits) {
              v.x += t[j].x; v.y += t[j].y; v.z += t[j].z; v.w += t[j].w;
            }
        }
        v.x = as_output(v.x, round_sum); v.y = as_output(v.y, round_sum);
        v.z = as_output(v.z, round_sum); v.w = as_output(v.w, round_sum);
      }
      if (pairs != nullptr) {
        float4 e = make_float4(0.f, 0.f, 0.f, 0.f);
        for (int k0 = 0; k0 < top; k0 += 8) {
          float4 t[8];
#pragma unroll
          for (int j = 0; j < 8; ++j)
            if (k0 + j < top) t[j] = *reinterpret_cast<const float4*>(pairs + (n * top + k0 + j) * width + c);
#pragma unroll
          for (int j = 0; j < 8; ++j)
            if (k0 + j < top) {
              e.x += t[j].x; e.y += t[j].y; e.z += t[j].z; e.w += t[j].w;
            }
        }
        v.x = fmaf(pair_weight, e.x, v.x); v.y = fmaf(pair_weight, e.y, v.y);
        v.z = fmaf(pair_weight, e.z, v.z); v.w = fmaf(pair_weight, e.w, v.w);
      }
      *reinterpret_cast<float4*>(row + c) = v;
      ss = fmaf(v.x, v.x, fmaf(v.y, v.y, fmaf(v.z, v.z, fmaf(v.w, v.w, ss))));
    }
  } else {
    for (int c = threadIdx.x; c < width; c += blockDim.x) {
      float v = 0.f;
      if (src != nullptr) {
        for (int s = 0; s < n_splits; ++s) v += to_f32<TS>(src[s * split_stride + n * width + c]);
        v = as_output(v, round_sum);
      }
      if (pairs != nullptr) {
        float e = 0.f;
        for (int k = 0; k < top; ++k) e += pairs[(n * top + k) * width + c];
        v = fmaf(pair_weight, e, v);
      }
      row[c] = v;
      ss = fmaf(v, v, ss);
    }
  }
  const float total = block_sum(ss, scratch);
  const float inv = 1.f / sqrtf(total / static_cast<float>(width) + eps);
  if (VEC) {
    for (int c = 4 * threadIdx.x; c < width; c += 4 * blockDim.x) {
      const float4 wv = na_load4<TW>(w + c), b = *reinterpret_cast<const float4*>(row + c);
      const float off = unit_offset ? 1.f : 0.f;
      float4 r = *reinterpret_cast<const float4*>(residual + n * width + c);
      r.x += b.x * inv * (wv.x + off); r.y += b.y * inv * (wv.y + off);
      r.z += b.z * inv * (wv.z + off); r.w += b.w * inv * (wv.w + off);
      *reinterpret_cast<float4*>(residual + n * width + c) = r;
      if (out != nullptr)
        *reinterpret_cast<uint2*>(out + n * width + c) = make_uint2(pack_bf16x2(r.x, r.y), pack_bf16x2(r.z, r.w));
    }
    return;
  }
  for (int c = threadIdx.x; c < width; c += blockDim.x) {
    const float wv = to_f32<TW>(w[c]) + (unit_offset ? 1.f : 0.f);
    const float r = residual[n * width + c] + row[c] * inv * wv;
    residual[n * width + c] = r;
    if (out != nullptr) out[n * width + c] = from_f32<TO>(r);
  }
}

// rows of a float32 stream rounded to the activation dtype (what the first branch of a model reads)
template <typename TO>
__global__ void round_rows_kernel(const float* __restrict__ x, TO* __restrict__ out, size_t total) {
  for (size_t i = blockIdx.x * static_cast<size_t>(blockDim.x) + threadIdx.x; i < total;
       i += static_cast<size_t>(gridDim.x) * blockDim.x)
    out[i] = from_f32<TO>(x[i]);
}

extern "C" int yk_round_rows(const float* x, void* out, int out_dtype, size_t total, hipStream_t stream) {
  if (total == 0) return 0;
  YK_REQUIRE(out_dtype == YK_BF16, "round_rows: the narrow dtype is bfloat16");
  const int grid = static_cast<int>(std::min<size_t>((total + 255) / 256, 65535));
  round_rows_kernel<bf16_t><<<grid, 256, 0, stream>>>(x, static_cast<bf16_t*>(out), total);
  return yk_check_launch("round_rows");
}

extern "C" int yk_norm_add(float* residual, const void* src, int src_dtype, int n_splits, int round_sum,
                           const float* pairs, int top, float pair_weight, const void* w, int w_dtype,
                           int unit_offset, float eps, void* out, int out_dtype, int n_rows, int width,
                           hipStream_t stream) {
  YK_REQUIRE(n_rows >= 0 && width > 0, "norm_add: bad sizes");
  YK_REQUIRE(src != nullptr || pairs != nullptr, "norm_add: no branch given");
  YK_REQUIRE(n_splits >= 1 && (n_splits == 1 || src_dtype == YK_F32), "norm_add: unreduced slices must be float32");
  YK_REQUIRE(pairs == nullptr || top >= 1, "norm_add: expert rows need a count per token");
  YK_REQUIRE(width <= 15 * 1024, "norm_add: rows of more than 15,360 elements do not fit the row buffer");
  YK_REQUIRE(out == nullptr || out_dtype == YK_BF16, "norm_add: the rounded copy is bfloat16");
  if (n_rows == 0) return 0;
  const size_t stride = static_cast<size_t>(n_rows) * width;
  const size_t lds = (static_cast<size_t>(width) + 17) * sizeof(float);
  auto al = [](const void* p) { return reinterpret_cast<uintptr_t>(p) % 16 == 0; };
  const bool vec = width % 4 == 0 && al(residual) && al(src) && al(pairs) && al(w) && al(out);
#define YK_CASE(SD, TS, WD, TW)                                                                            \
  if ((src == nullptr || src_dtype == SD) && w_dtype == WD) {                                                \
    if (vec)                                                                                                 \
      norm_add_kernel<TS, TW, bf16_t, true><<<n_rows, 256, lds, stream>>>(                                   \
          residual, static_cast<const TS*>(src), n_splits, stride, round_sum, pairs, top, pair_weight,       \
          static_cast<const TW*>(w), unit_offset, eps, static_cast<bf16_t*>(out), width);                    \
    else                                                                                                     \
      norm_add_kernel<TS, TW, bf16_t, false><<<n_rows, 256, lds, stream>>>(                                  \
          residual, static_cast<const TS*>(src), n_splits, stride, round_sum, pairs, top, pair_weight,       \
          static_cast<const TW*>(w), unit_offset, eps, static_cast<bf16_t*>(out), width);                    \
    return yk_check_launch("norm_add");                                                                      \
  }
  YK_CASE(YK_F32, float, YK_F32, float)
  YK_CASE(YK_F32, float, YK_BF16, bf16_t)
  YK_CASE(YK_BF16, bf16_t, YK_F32, float)
  YK_CASE(YK_BF16, bf16_t, YK_BF16, bf16_t)
#undef YK_CASE
  return yk_fail("norm_add: unsupported dtype combination");
}

// ------------------------------------------------------------- the stream normed after the sum
//   b        = branch_scale * (a-term + b-term) * channel weight
//   r        = residual_scale * residual[n, :] + b
//   residual = r / sqrt(mean(r^2) + eps) * w'           (w' = w or 1 + w), and its rounded copy beside it
// A term is a branch's rows (activation dtype, float32, or a product's unreduced slices), as they are or first divided
// by their own root mean square and multiplied by a weight; the second term and the channel weight may be absent.  Both
// terms' sums of squares are reduced together.  One workgroup a row; rows of up to 4,096 elements stay in registers
// between the reductions (VEC: four columns a thread and piece, everything asked for before the first reduction), longer
// or odd ones in LDS.
struct SumTerm {
  const void* src;
  int bf16;  // 1: bfloat16 rows; 0: float32 rows or slices
  int n_splits;
  int round_sum;
  float eps;
  const void* w;  // null: added as it is
};

__device__ __forceinline__ void block_sum2(float& a, float& b, float* scratch) {
  a = wave_sum(a);
  b = wave_sum(b);
  const int wave = threadIdx.x / kWave, lane = threadIdx.x % kWave, n_waves = blockDim.x / kWave;
  __syncthreads();  // scratch may still be read from an earlier call
  if (lane == 0) scratch[2 * wave] = a, scratch[2 * wave + 1] = b;
  __syncthreads();
  a = b = 0.f;
  for (int i = 0; i < n_waves; ++i) a += scratch[2 * i], b += scratch[2 * i + 1];
}

__device__ __forceinline__ float4 sum_term4(const SumTerm& t, size_t at, size_t stride) {
  float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
  if (t.bf16) {
    v = na_load4<bf16_t>(static_cast<const bf16_t*>(t.src) + at);
  } else {
    const float* p = static_cast<const float*>(t.src) + at;
    for (int s0 = 0; s0 < t.n_splits; s0 += 8) {
      float4 x[8];
#pragma unroll
      for (int j = 0; j < 8; ++j)
        if (s0 + j < t.n_splits) x[j] = *reinterpret_cast<const float4*>(p + (s0 + j) * stride);
#pragma unroll
      for (int j = 0; j < 8; ++j)
        if (s0 + j < t.n_splits) {
          v.x += x[j].x; v.y += x[j].y; v.z += x[j].z; v.w += x[j].w;
        }
    }
    v = make_float4(as_output(v.x, t.round_sum), as_output(v.y, t.round_sum), as_output(v.z, t.round_sum), as_output(v.w, t.round_sum));
  }
  return v;
}

__device__ __forceinline__ float sum_term1(const SumTerm& t, size_t at, size_t stride) {
  if (t.bf16) return to_f32<bf16_t>(static_cast<const bf16_t*>(t.src)[at]);
  float v = 0.f;
  for (int s = 0; s < t.n_splits; ++s) v += static_cast<const float*>(t.src)[at + s * stride];
  return as_output(v, t.round_sum);
}

__device__ __forceinline__ float dot4(float4 v) { return fmaf(v.x, v.x, fmaf(v.y, v.y, fmaf(v.z, v.z, v.w * v.w))); }
__device__ __forceinline__ float4 mul4(float4 a, float4 b) { return make_float4(a.x * b.x, a.y * b.y, a.z * b.z, a.w * b.w); }
__device__ __forceinline__ float4 scaled4(float4 a, float s) { return make_float4(a.x * s, a.y * s, a.z * s, a.w * s); }

// P: pieces of 4 columns x blockDim.x a thread holds
template <typename TW, int P>
__global__ __launch_bounds__(256) void sum_norm_vec_kernel(float* __restrict__ residual, SumTerm ta, SumTerm tb, int has_b,
                                                           size_t stride, float branch_scale, const TW* __restrict__ cw,
                                                           float residual_scale, const TW* __restrict__ w, int unit_offset,
                                                           float eps, bf16_t* __restrict__ out, int width) {
  __shared__ float scratch[34];
  const size_t n = blockIdx.x;
  const float4 one = make_float4(1.f, 1.f, 1.f, 1.f), zero = make_float4(0.f, 0.f, 0.f, 0.f);
  float4 a[P], b[P], rs[P], wn[P], wc[P], wa[P], wb[P];
  float sa = 0.f, sb = 0.f;
#pragma unroll
  for (int k = 0; k < P; ++k) {
    const int c = 4 * (threadIdx.x + blockDim.x * k);
    a[k] = b[k] = rs[k] = wn[k] = zero;
    wc[k] = wa[k] = wb[k] = one;
    if (c >= width) continue;
    const size_t at = n * width + c;
    rs[k] = *reinterpret_cast<const float4*>(residual + at);
    wn[k] = na_load4<TW>(w + c);
    if (cw != nullptr) wc[k] = na_load4<TW>(cw + c);
    if (ta.w != nullptr) wa[k] = na_load4<TW>(static_cast<const TW*>(ta.w) + c);
    if (has_b && tb.w != nullptr) wb[k] = na_load4<TW>(static_cast<const TW*>(tb.w) + c);
    a[k] = sum_term4(ta, at, stride);
    if (has_b) b[k] = sum_term4(tb, at, stride);
  }
#pragma unroll
  for (int k = 0; k < P; ++k) sa += dot4(a[k]), sb += dot4(b[k]);
  float ia = 1.f, ib = 1.f;
  if (ta.w != nullptr || (has_b && tb.w != nullptr)) {
    block_sum2(sa, sb, scratch);
    if (ta.w != nullptr) ia = 1.f / sqrtf(sa / static_cast<float>(width) + ta.eps);
    if (has_b && tb.w != nullptr) ib = 1.f / sqrtf(sb / static_cast<float>(width) + tb.eps);
  }
  float ss = 0.f, none = 0.f;
#pragma unroll
  for (int k = 0; k < P; ++k) {
    float4 v = scaled4(mul4(a[k], wa[k]), ia);
    if (has_b) {
      const float4 u = mul4(b[k], wb[k]);
      v = make_float4(fmaf(u.x, ib, v.x), fmaf(u.y, ib, v.y), fmaf(u.z, ib, v.z), fmaf(u.w, ib, v.w));
    }
    v = mul4(scaled4(v, branch_scale), wc[k]);
    rs[k] = make_float4(fmaf(residual_scale, rs[k].x, v.x), fmaf(residual_scale, rs[k].y, v.y), fmaf(residual_scale, rs[k].z, v.z),
                        fmaf(residual_scale, rs[k].w, v.w));
    if (4 * (threadIdx.x + static_cast<int>(blockDim.x) * k) < width) ss += dot4(rs[k]);
  }
  block_sum2(ss, none, scratch);
  const float inv = 1.f / sqrtf(ss / static_cast<float>(width) + eps);
  const float off = unit_offset ? 1.f : 0.f;
#pragma unroll
  for (int k = 0; k < P; ++k) {
    const int c = 4 * (threadIdx.x + blockDim.x * k);
    if (c >= width) continue;
    const float4 r = make_float4(rs[k].x * inv * (wn[k].x + off), rs[k].y * inv * (wn[k].y + off), rs[k].z * inv * (wn[k].z + off),
                                 rs[k].w * inv * (wn[k].w + off));
    *reinterpret_cast<float4*>(residual + n * width + c) = r;
    if (out != nullptr) *reinterpret_cast<uint2*>(out + n * width + c) = make_uint2(pack_bf16x2(r.x, r.y), pack_bf16x2(r.z, r.w));
  }
}

template <typename TW>
__global__ __launch_bounds__(256) void sum_norm_kernel(float* __restrict__ residual, SumTerm ta, SumTerm tb, int has_b, size_t stride,
                                                       float branch_scale, const TW* __restrict__ cw, float residual_scale,
                                                       const TW* __restrict__ w, int unit_offset, float eps,
                                                       bf16_t* __restrict__ out, int width) {
  extern __shared__ float row[];  // [width] (and [width] for a second term), then 34 floats of scratch
  float* second = row + width;
  float* scratch = row + (has_b ? 2 : 1) * static_cast<size_t>(width);
  const size_t n = blockIdx.x;
  float sa = 0.f, sb = 0.f;
  for (int c = threadIdx.x; c < width; c += blockDim.x) {  // (every thread keeps to its own columns throughout)
    const float a = sum_term1(ta, n * width + c, stride);
    row[c] = a;
    sa = fmaf(a, a, sa);
    if (has_b) {
      const float b = sum_term1(tb, n * width + c, stride);
      second[c] = b;
      sb = fmaf(b, b, sb);
    }
  }
  block_sum2(sa, sb, scratch);
  const float ia = ta.w != nullptr ? 1.f / sqrtf(sa / static_cast<float>(width) + ta.eps) : 1.f;
  const float ib = has_b && tb.w != nullptr ? 1.f / sqrtf(sb / static_cast<float>(width) + tb.eps) : 1.f;
  float ss = 0.f, none = 0.f;
  for (int c = threadIdx.x; c < width; c += blockDim.x) {
    float v = row[c] * (ta.w != nullptr ? to_f32<TW>(static_cast<const TW*>(ta.w)[c]) : 1.f) * ia;
    if (has_b) v = fmaf(second[c] * (tb.w != nullptr ? to_f32<TW>(static_cast<const TW*>(tb.w)[c]) : 1.f), ib, v);
    v *= branch_scale;
    if (cw != nullptr) v *= to_f32<TW>(cw[c]);
    const float r = fmaf(residual_scale, residual[n * width + c], v);
    row[c] = r;
    ss = fmaf(r, r, ss);
  }
  block_sum2(ss, none, scratch);
  const float inv = 1.f / sqrtf(ss / static_cast<float>(width) + eps);
  for (int c = threadIdx.x; c < width; c += blockDim.x) {
    const float r = row[c] * inv * (to_f32<TW>(w[c]) + (unit_offset ? 1.f : 0.f));
    residual[n * width + c] = r;
    if (out != nullptr) out[n * width + c] = f32_to_bf16(r);
  }
}

// Terms a and b (b_src null: one term): dtype, slices, whether their sum is rounded, eps and weight (null: as it is).
// All weights share w_dtype.
extern "C" int yk_sum_norm(float* residual, const void* a_src, int a_dtype, int a_splits, int a_round, float a_eps, const void* a_w,
                           const void* b_src, int b_dtype, int b_splits, int b_round, float b_eps, const void* b_w,
                           float branch_scale, const void* channel_w, float residual_scale, const void* w, int w_dtype,
                           int unit_offset, float eps, void* out, int n_rows, int width, hipStream_t stream) {
  YK_REQUIRE(n_rows >= 0 && width > 0 && residual != nullptr && w != nullptr, "sum_norm: bad sizes");
  YK_REQUIRE(a_src != nullptr, "sum_norm: no branch given");
  YK_REQUIRE(a_splits >= 1 && (a_splits == 1 || a_dtype == YK_F32) && (b_src == nullptr || (b_splits >= 1 && (b_splits == 1 || b_dtype == YK_F32))),
             "sum_norm: unreduced slices must be float32");
  YK_REQUIRE((b_src != nullptr ? 2 : 1) * static_cast<long>(width) <= 15 * 1024, "sum_norm: the rows do not fit the row buffer");
  if (n_rows == 0) return 0;
  const size_t stride = static_cast<size_t>(n_rows) * width;
  const SumTerm ta{a_src, a_dtype == YK_BF16, a_splits, a_round, a_eps, a_w};
  const SumTerm tb{b_src, b_dtype == YK_BF16, b_splits, b_round, b_eps, b_w};
  const int has_b = b_src != nullptr;
  auto al = [](const void* p) { return reinterpret_cast<uintptr_t>(p) % 16 == 0; };
  const bool vec = width % 4 == 0 && width <= 4096 && al(residual) && al(a_src) && al(b_src) && al(a_w) && al(b_w) && al(channel_w) &&
                   al(w) && al(out);
#define YK_ARGS(TW)                                                                                                        \
  residual, ta, tb, has_b, stride, branch_scale, static_cast<const TW*>(channel_w), residual_scale, static_cast<const TW*>(w), \
      unit_offset, eps, static_cast<bf16_t*>(out), width
#define YK_CASE(WD, TW)                                                                                                    \
  if (w_dtype == WD) {                                                                                                     \
    if (vec && width <= 1024)                                                                                              \
      sum_norm_vec_kernel<TW, 1><<<n_rows, 256, 0, stream>>>(YK_ARGS(TW));                                                 \
    else if (vec && width <= 2048)                                                                                         \
      sum_norm_vec_kernel<TW, 2><<<n_rows, 256, 0, stream>>>(YK_ARGS(TW));                                                 \
    else if (vec)                                                                                                          \
      sum_norm_vec_kernel<TW, 4><<<n_rows, 256, 0, stream>>>(YK_ARGS(TW));                                                 \
    else                                                                                                                   \
      sum_norm_kernel<TW><<<n_rows, 256, ((has_b ? 2 : 1) * static_cast<size_t>(width) + 34) * sizeof(float), stream>>>(YK_ARGS(TW)); \
    return yk_check_launch("sum_norm");                                                                                    \
  }
  YK_CASE(YK_F32, float)
  YK_CASE(YK_BF16, bf16_t)
#undef YK_CASE
#undef YK_ARGS
  return yk_fail("sum_norm: unsupported weight dtype");
}
