// Inputs mixed with the token before's, and the small second product of a low-rank pair.
//
//   token_shift_mix: out[s, n, :] = x[n, :] + (x'[n, :] - x[n, :]) * mu[s, :]   for several mixes s at once
//
// x' is the row of the token before in the same request: the batch's row n - 1 inside a span, the request's state
// (zeros before its first token) for a span's first token.  The thread that reads the state for its columns is also the
// one that leaves the span's last row there, so a step needs no second pass.  The mix is float32, rounded once.
//
//   low_rank: z[n, c] = sum_j act(y[n, j]) * w[c, j]    float32, for few tokens and a rank of up to a few hundred
//
//   act_rows: out[n, j] = act(y[n, j]) for rows with a stride, rounded once (what a product of many rows reads)
#include <algorithm>

#include "common.h"

template <typename T>
__device__ __forceinline__ float4 tm_load4(const T* p) {
  if constexpr (sizeof(T) == 2) {
    const uint2 w = *reinterpret_cast<const uint2*>(p);
    return make_float4(__uint_as_float(w.x << 16), __uint_as_float(w.x & 0xffff0000u), __uint_as_float(w.y << 16),
                       __uint_as_float(w.y & 0xffff0000u));
  } else {
    return *reinterpret_cast<const float4*>(p);
  }
}
template <typename T>
__device__ __forceinline__ void tm_store4(T* p, float4 v) {
  if constexpr (sizeof(T) == 2)
    *reinterpret_cast<uint2*>(p) = make_uint2(pack_bf16x2(v.x, v.y), pack_bf16x2(v.z, v.w));
  else
    *reinterpret_cast<float4*>(p) = v;
}

constexpr int kMaxMixes = 8;

template <typename T, bool VEC>
__global__ __launch_bounds__(256) void token_shift_mix_kernel(const T* __restrict__ x, const float* __restrict__ mu, int n_mixes,
                                                              T* state, const int32_t* __restrict__ token_seq,
                                                              const int32_t* __restrict__ seq_qstart,
                                                              const int32_t* __restrict__ seq_qlen,
                                                              const int32_t* __restrict__ state_slots, T* __restrict__ out,
                                                              int width, int n_tokens) {
  constexpr int E = VEC ? 4 : 1;
  const int per_row = width / E;  // (VEC: the width is a multiple of four)
  const size_t total = static_cast<size_t>(n_tokens) * per_row, mix_stride = static_cast<size_t>(n_tokens) * width;
  for (size_t i = blockIdx.x * static_cast<size_t>(blockDim.x) + threadIdx.x; i < total; i += static_cast<size_t>(gridDim.x) * blockDim.x) {
    const int n = static_cast<int>(i / per_row), c = static_cast<int>(i % per_row) * E;
    const int seq = token_seq[n], q0 = seq_qstart[seq];
    const size_t at = static_cast<size_t>(n) * width + c;
    T* st = state + static_cast<size_t>(state_slots[seq]) * width + c;
    if constexpr (VEC) {
      const float4 now = tm_load4<T>(x + at);
      const float4 was = n == q0 ? tm_load4<T>(st) : tm_load4<T>(x + at - width);
      if (n == q0) tm_store4<T>(st, tm_load4<T>(x + static_cast<size_t>(q0 + seq_qlen[seq] - 1) * width + c));
      const float4 d = make_float4(was.x - now.x, was.y - now.y, was.z - now.z, was.w - now.w);
      for (int s = 0; s < n_mixes; ++s) {
        const float4 m = *reinterpret_cast<const float4*>(mu + static_cast<size_t>(s) * width + c);
        tm_store4<T>(out + s * mix_stride + at, make_float4(fmaf(d.x, m.x, now.x), fmaf(d.y, m.y, now.y), fmaf(d.z, m.z, now.z), fmaf(d.w, m.w, now.w)));
      }
    } else {
      const float now = to_f32<T>(x[at]);
      const float was = to_f32<T>(n == q0 ? *st : x[at - width]);
      if (n == q0) *st = x[static_cast<size_t>(q0 + seq_qlen[seq] - 1) * width + c];
      for (int s = 0; s < n_mixes; ++s) out[s * mix_stride + at] = from_f32<T>(fmaf(was - now, mu[static_cast<size_t>(s) * width + c], now));
    }
  }
}

extern "C" int yk_token_shift_mix(const void* x, int dtype, const float* mu, int n_mixes, void* state, const int32_t* token_seq,
                                  const int32_t* seq_qstart, const int32_t* seq_qlen, const int32_t* state_slots, void* out,
                                  int n_tokens, int width, hipStream_t stream) {
  YK_REQUIRE(n_tokens >= 0 && width > 0 && n_mixes >= 1 && n_mixes <= kMaxMixes, "token_shift_mix: bad sizes");
  YK_REQUIRE(state != nullptr && mu != nullptr, "token_shift_mix: the state or the mixes are missing");
  if (n_tokens == 0) return 0;
  auto al16 = [](const void* p) { return reinterpret_cast<uintptr_t>(p) % 16 == 0; };
  const bool vec = width % 4 == 0 && al16(x) && al16(mu) && al16(state) && al16(out);
  const size_t total = static_cast<size_t>(n_tokens) * (vec ? width / 4 : width);
  const int grid = static_cast<int>(std::min<size_t>((total + 255) / 256, 1 << 20));
#define YK_CASE(D, T, V)                                                                                                          \
  if (dtype == D && vec == V) {                                                                                                   \
    token_shift_mix_kernel<T, V><<<grid, 256, 0, stream>>>(static_cast<const T*>(x), mu, n_mixes, static_cast<T*>(state), token_seq, \
                                                           seq_qstart, seq_qlen, state_slots, static_cast<T*>(out), width, n_tokens); \
    return yk_check_launch("token_shift_mix");                                                                                    \
  }
  YK_CASE(YK_F32, float, true)
  YK_CASE(YK_F32, float, false)
  YK_CASE(YK_BF16, bf16_t, true)
  YK_CASE(YK_BF16, bf16_t, false)
#undef YK_CASE
  return yk_fail("token_shift_mix: unsupported dtype");
}

// act: 0 none, 1 tanh
__device__ __forceinline__ float low_rank_act(float v, int act) { return act == 1 ? tanhf(v) : v; }

constexpr int kLowRankTokens = 8;  // tokens a workgroup takes at a time

// a workgroup: up to eight tokens, their rows of y in LDS (padded with zeros to a multiple of eight).  VEC (a rank that is a
// multiple of eight): eight lanes a column, each taking pieces of eight of its row of w for all the tokens, so that a column's
// row is read in one round trip and in consecutive bytes; the sums meet by exchanges and lane t stores token t's.  Otherwise a
// thread a column.
template <typename T, typename TW, bool VEC>
__global__ __launch_bounds__(256) void low_rank_kernel(const T* __restrict__ y, int y_stride, const TW* __restrict__ w, int act,
                                                       float* __restrict__ out, int n_tokens, int cols, int rank) {
  extern __shared__ float rows[];  // [kLowRankTokens][rp]
  const int rp = (rank + 7) / 8 * 8;
  const int n0 = blockIdx.y * kLowRankTokens, live = min(kLowRankTokens, n_tokens - n0);
  for (int i = threadIdx.x; i < kLowRankTokens * rp; i += blockDim.x) {
    const int t = i / rp, j = i % rp;
    rows[i] = t < live && j < rank ? low_rank_act(to_f32<T>(y[static_cast<size_t>(n0 + t) * y_stride + j]), act) : 0.f;
  }
  __syncthreads();
  float acc[kLowRankTokens];
#pragma unroll
  for (int t = 0; t < kLowRankTokens; ++t) acc[t] = 0.f;
  if (VEC) {
    const int sub = threadIdx.x % 8, c = blockIdx.x * (blockDim.x / 8) + threadIdx.x / 8;
    const TW* wr = w + static_cast<size_t>(min(c, cols - 1)) * rank;  // (a column beyond the last works on it and stores nothing)
    for (int j = 8 * sub; j < rank; j += 64) {
      const float4 a = tm_load4<TW>(wr + j), b = tm_load4<TW>(wr + j + 4);
#pragma unroll
      for (int t = 0; t < kLowRankTokens; ++t) {
        const float4 p = *reinterpret_cast<const float4*>(rows + t * rp + j), q = *reinterpret_cast<const float4*>(rows + t * rp + j + 4);
        acc[t] = fmaf(a.x, p.x, fmaf(a.y, p.y, fmaf(a.z, p.z, fmaf(a.w, p.w, fmaf(b.x, q.x, fmaf(b.y, q.y, fmaf(b.z, q.z, fmaf(b.w, q.w, acc[t]))))))));
      }
    }
    float mine = 0.f;
#pragma unroll
    for (int t = 0; t < kLowRankTokens; ++t) {
#pragma unroll
      for (int o = 4; o > 0; o >>= 1) acc[t] += __shfl_xor(acc[t], o, 8);
      if (t == sub) mine = acc[t];
    }
    if (c < cols && sub < live) out[static_cast<size_t>(n0 + sub) * cols + c] = mine;
    return;
  }
  const int c = blockIdx.x * blockDim.x + threadIdx.x;
  if (c >= cols) return;
  const TW* wr = w + static_cast<size_t>(c) * rank;
  for (int j = 0; j < rank; ++j) {
    const float a = to_f32<TW>(wr[j]);
#pragma unroll
    for (int t = 0; t < kLowRankTokens; ++t) acc[t] = fmaf(a, rows[t * rp + j], acc[t]);
  }
#pragma unroll
  for (int t = 0; t < kLowRankTokens; ++t)
    if (t < live) out[static_cast<size_t>(n0 + t) * cols + c] = acc[t];
}

extern "C" int yk_low_rank(const void* y, int y_stride, int y_dtype, const void* w, int w_dtype, int act, float* out, int n_tokens,
                           int cols, int rank, hipStream_t stream) {
  YK_REQUIRE(n_tokens >= 0 && cols > 0 && rank > 0 && y_stride >= rank, "low_rank: bad sizes");
  YK_REQUIRE(act == 0 || act == 1, "low_rank: unknown activation");
  YK_REQUIRE(rank <= 1536, "low_rank: ranks of more than 1,536 do not fit the row buffer");
  YK_REQUIRE((n_tokens + kLowRankTokens - 1) / kLowRankTokens <= 65535, "low_rank: too many tokens for one launch");
  if (n_tokens == 0) return 0;
  const bool vec = rank % 8 == 0 && reinterpret_cast<uintptr_t>(w) % 16 == 0;
  const int columns = vec ? 32 : 256;  // of a workgroup
  dim3 grid((cols + columns - 1) / columns, (n_tokens + kLowRankTokens - 1) / kLowRankTokens);
  const size_t lds = static_cast<size_t>(kLowRankTokens) * ((rank + 7) / 8 * 8) * sizeof(float);
#define YK_CASE(YD, T, WD, TW, V)                                                                                    \
  if (y_dtype == YD && w_dtype == WD && vec == V) {                                                                  \
    low_rank_kernel<T, TW, V><<<grid, 256, lds, stream>>>(static_cast<const T*>(y), y_stride, static_cast<const TW*>(w), act, out, \
                                                          n_tokens, cols, rank);                                     \
    return yk_check_launch("low_rank");                                                                              \
  }
  YK_CASE(YK_F32, float, YK_F32, float, true)
  YK_CASE(YK_F32, float, YK_F32, float, false)
  YK_CASE(YK_BF16, bf16_t, YK_BF16, bf16_t, true)
  YK_CASE(YK_BF16, bf16_t, YK_BF16, bf16_t, false)
  YK_CASE(YK_BF16, bf16_t, YK_F32, float, true)
  YK_CASE(YK_BF16, bf16_t, YK_F32, float, false)
#undef YK_CASE
  return yk_fail("low_rank: unsupported dtype combination");
}

template <typename T>
__global__ void act_rows_kernel(const T* __restrict__ y, int y_stride, int act, T* __restrict__ out, int cols, size_t total) {
  for (size_t i = blockIdx.x * static_cast<size_t>(blockDim.x) + threadIdx.x; i < total; i += static_cast<size_t>(gridDim.x) * blockDim.x)
    out[i] = from_f32<T>(low_rank_act(to_f32<T>(y[(i / cols) * y_stride + i % cols]), act));
}

extern "C" int yk_act_rows(const void* y, int y_stride, int dtype, int act, void* out, int n_tokens, int cols, hipStream_t stream) {
  YK_REQUIRE(n_tokens >= 0 && cols > 0 && y_stride >= cols, "act_rows: bad sizes");
  YK_REQUIRE(act == 0 || act == 1, "act_rows: unknown activation");
  const size_t total = static_cast<size_t>(n_tokens) * cols;
  if (total == 0) return 0;
  const int grid = static_cast<int>(std::min<size_t>((total + 255) / 256, 1 << 20));
  if (dtype == YK_F32)
    act_rows_kernel<float><<<grid, 256, 0, stream>>>(static_cast<const float*>(y), y_stride, act, static_cast<float*>(out), cols, total);
  else if (dtype == YK_BF16)
    act_rows_kernel<bf16_t><<<grid, 256, 0, stream>>>(static_cast<const bf16_t*>(y), y_stride, act, static_cast<bf16_t*>(out), cols, total);
  else
    return yk_fail("act_rows: unsupported dtype");
  return yk_check_launch("act_rows");
}
