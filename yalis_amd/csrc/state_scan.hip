// Recurrences whose memory is a matrix per head, S [dim][vdim] float32 in the request's state slot:
//
//   S <- diag(a_t) S                       a_t: one decay for the head, or one per key channel (row of S)
//   u  = v_t                               plain write
//   u  = beta_t (v_t - S^T k_t)            delta rule
//   u  = dt_t v_t                          a write as strong as the token's step (state-space duality: with the head's
//                                          decay exp(-exp(A_log) dt_t), dt_t = softplus(x + dt_bias), q = C, k = B)
//   S <- S + k_t u^T,   o_t = S^T q_t      (the read-out sees the token's own write; + skip_h v_t where a skip is given)
// or, with a bonus b per head and key channel, the read-out of the memory as it was before the token:
//   o_t = (S + diag(b) k_t v_t^T)^T q_t,   S <- diag(a_t) S + k_t v_t^T
//
// The columns of S never meet: column e needs k_t, q_t, a_t, beta_t and its own v_t[e] only.  So a
// column lives in the registers of a group of TPC lanes (lane s of the group holds the rows s,
// 16 s .. 16 s + 15), the two sums over rows are exchanges inside the group, and a workgroup walks a
// request's span token by token with k, q and the decays of the next 32 tokens staged in LDS (a wave
// per token and vector makes the unit norm while it stages), read back 16 bytes at a time.  Decays, write strengths and unit norms are made here, in float32, from the
// projections' raw outputs:
//   decay per head:     exp(-exp(A_log[h]) * softplus(x[n, h] + dt_bias[h]))
//   decay per channel:  sigmoid(z[n, h, i] + bias[h, i]) ^ (1 / tau)  =  exp(logsigmoid(.) / tau), or
//                       exp(-exp(A_log[h]) * softplus(z[n, h, i] + dt_bias[h, i])), or exp(-exp(z[n, h, i] + bias[h, i]))
//  fixed decay:        a constant of the model per head
//   beta:               sigmoid(x[n, h])
//   unit vectors:       q / sqrt(sum q^2 + eps), k likewise (with unit_eps >= 0), then q * q_scale
// A span cut anywhere gives the same S bit for bit: every token's step is made alone.
//
// Beside it: the read-out's norm and gate (each head's o divided by its root mean square, times a
// weight shared by the heads, times silu or the sigmoid of a gate column), and the shift of a convolution's kept
// inputs by a span.
#include <algorithm>

#include "common.h"

constexpr int kScanRowsMax = 16;  // rows of S a lane holds at the most (template R: 8 or 16): sub * R .. sub * R + R - 1 of its column
constexpr int kScanTokens = 32;  // tokens staged at a time (fewer where LDS would not hold them)

__device__ __forceinline__ float scan_softplus(float x) { return fmaxf(x, 0.f) + log1pf(expf(-fabsf(x))); }

// a decay per key channel from its biased logit x: kinds 1, 2 and 3 of yk_linear_state_scan
__device__ __forceinline__ float channel_decay(float x, int mode, float tau, float rate) {
  if (mode == 1) return expf(-scan_softplus(-x) / tau);
  if (mode == 2) return expf(-rate * scan_softplus(x));
  return expf(-expf(x));
}

// the sum over the TPC lanes of a column (lanes that differ in their low bits), in all of them.  Inside
// a row of 16 lanes the exchanges are register moves (quad permutations, then rotations of the row by 4
// and by 8: after the quads' sums, s_j = Q_j + Q_(j+1) and s_j + s_(j+2) is the row's sum); wider groups
// go on through the LDS pipe.
__device__ __forceinline__ float dpp_add(float v, int ctrl_xor1_2_ror4_8) {
  const int x = __float_as_int(v);
  int y;
  switch (ctrl_xor1_2_ror4_8) {
    case 0: y = __builtin_amdgcn_update_dpp(0, x, 0xB1, 0xf, 0xf, false); break;   // quad_perm [1,0,3,2]
    case 1: y = __builtin_amdgcn_update_dpp(0, x, 0x4E, 0xf, 0xf, false); break;   // quad_perm [2,3,0,1]
    case 2: y = __builtin_amdgcn_update_dpp(0, x, 0x124, 0xf, 0xf, false); break;  // row_ror:4
    default: y = __builtin_amdgcn_update_dpp(0, x, 0x128, 0xf, 0xf, false); break; // row_ror:8
  }
  return v + __int_as_float(y);
}
template <int TPC>
__device__ __forceinline__ float column_sum(float v) {
  if (TPC >= 2) v = dpp_add(v, 0);
  if (TPC >= 4) v = dpp_add(v, 1);
  if (TPC == 8) {
    // two quads a column: each takes the other's sum (quads 0 and 2 from four lanes up, 1 and 3 from four down)
    const int x = __float_as_int(v);
    int y = __builtin_amdgcn_update_dpp(0, x, 0x104, 0xf, 0x5, false);  // row_shl:4 into quads 0 and 2
    y = __builtin_amdgcn_update_dpp(y, x, 0x114, 0xf, 0xa, false);      // row_shr:4 into quads 1 and 3
    v += __int_as_float(y);
  }
  if (TPC >= 16) {
    v = dpp_add(v, 2);
    v = dpp_add(v, 3);
  }
  if (TPC >= 32) {  // lanes r and r + 16
    const auto a = __builtin_amdgcn_permlane16_swap(__float_as_uint(v), __float_as_uint(v), false, false);
    v = __uint_as_float(a[0]) + __uint_as_float(a[1]);
  }
  if (TPC >= 64) {  // and the other half of the wave
    const auto b = __builtin_amdgcn_permlane32_swap(__float_as_uint(v), __float_as_uint(v), false, false);
    v = __uint_as_float(b[0]) + __uint_as_float(b[1]);
  }
  return v;
}

// eight consecutive elements (16-byte aligned where T is bfloat16, 32 where float) as floats
template <typename T>
__device__ __forceinline__ void scan_load8(const T* p, float* out);
template <>
__device__ __forceinline__ void scan_load8<float>(const float* p, float* out) {
  const float4 a = *reinterpret_cast<const float4*>(p), b = *reinterpret_cast<const float4*>(p + 4);
  out[0] = a.x; out[1] = a.y; out[2] = a.z; out[3] = a.w; out[4] = b.x; out[5] = b.y; out[6] = b.z; out[7] = b.w;
}
template <>
__device__ __forceinline__ void scan_load8<bf16_t>(const bf16_t* p, float* out) {
  const uint4 w = *reinterpret_cast<const uint4*>(p);
  out[0] = __uint_as_float(w.x << 16); out[1] = __uint_as_float(w.x & 0xffff0000u);
  out[2] = __uint_as_float(w.y << 16); out[3] = __uint_as_float(w.y & 0xffff0000u);
  out[4] = __uint_as_float(w.z << 16); out[5] = __uint_as_float(w.z & 0xffff0000u);
  out[6] = __uint_as_float(w.w << 16); out[7] = __uint_as_float(w.w & 0xffff0000u);
}

// The general form: any sizes and alignments, every kind of decay, write and read-out chosen as it runs.
// LDS per staged token: k and q padded to TPC * 16 floats each (rows past dim are zeros, so nobody
// asks whether a row exists), the per-channel decays likewise where there are any
template <typename T, int TPC, int kScanRows>
__global__ __launch_bounds__(256) void linear_state_scan_kernel(
    const T* __restrict__ qkv, int qkv_stride, int n_heads, int n_kv, int dim, int vdim, float* __restrict__ state,
    const int32_t* __restrict__ seq_qstart, const int32_t* __restrict__ seq_qlen, const int32_t* __restrict__ state_slots,
    float q_scale, float unit_eps, int decay_mode, const float* __restrict__ decay, int decay_stride, int decay_col,
    const float* __restrict__ decay_p0, const float* __restrict__ decay_p1, float tau, const float* __restrict__ beta,
    int beta_stride, int beta_col, int chunk, float* __restrict__ out, int q_col, int k_col, int v_col, int write_mode,
    const float* __restrict__ skip, const T* __restrict__ beta_rows, const float* __restrict__ bonus) {
  extern __shared__ float lds[];
  constexpr int DP = TPC * kScanRows;  // padded key channels
  constexpr int DS = DP + 4;           // a staged row's stride: rows of different tokens then start in different banks
  const int cols_per_block = blockDim.x / TPC;
  float* ks = lds;                                        // [chunk][DS]
  float* qs = ks + chunk * DS;                            // [chunk][DS]
  float* as = qs + chunk * DS;                            // [chunk][DS] (per channel) or [chunk]
  const bool per_channel = decay_mode != 0 && decay_mode != 4;
  float* vs = as + chunk * (per_channel ? DS : 1);        // [chunk][cols_per_block]
  float* bs = vs + chunk * cols_per_block;                // [chunk]
  float* kqs = bs + chunk;                                // [chunk]: k . q (times the bonus) of every token, as they enter the recurrence
  float* us = kqs + chunk;                                // [DS]: the head's bonus, where there is one

  const int seq = blockIdx.x, h = blockIdx.y, kvh = h / (n_heads / n_kv);
  const int col0 = blockIdx.z * cols_per_block;
  const int sub = threadIdx.x % TPC, col_local = threadIdx.x / TPC, col = col0 + col_local;
  const bool has_col = col < vdim;
  const int wave = threadIdx.x / kWave, lane = threadIdx.x % kWave, n_waves = blockDim.x / kWave;
  const int q0 = seq_qstart[seq], ql = seq_qlen[seq];
  float* S_head = state + (static_cast<size_t>(state_slots[seq]) * n_heads + h) * dim * vdim;
  const bool delta = write_mode == 1;
  const float skip_h = skip != nullptr ? skip[h] : 0.f;
  const bool read_first = bonus != nullptr;  // the read-out sees the memory as it was
  if (read_first)
    for (int i = threadIdx.x; i < DP; i += blockDim.x) us[i] = i < dim ? bonus[h * dim + i] : 0.f;
  // per channel: the vector that joins the logits, and (kind 2) what the softplus is multiplied with
  const float* dec_bias = decay_mode == 2 ? decay_p1 : decay_p0;
  const float dec_rate = decay_mode == 2 ? expf(decay_p0[h]) : 1.f;

  float S[kScanRows];
#pragma unroll
  for (int r = 0; r < kScanRows; ++r) {
    const int i = sub * kScanRows + r;
    S[r] = has_col && i < dim ? S_head[static_cast<size_t>(i) * vdim + col] : 0.f;
  }
  for (int t0 = 0; t0 < ql; t0 += chunk) {
    const int nt = min(chunk, ql - t0);
    __syncthreads();  // the chunk before has been read
    // q and k of the chunk's tokens to LDS, every load of a thread asked for before the first is used
    // (one after the other they cost a round trip to memory each)
    {
      const float q_mul = unit_eps >= 0.f ? 1.f : q_scale;
      const int total = 2 * nt * DP;
      for (int i0 = threadIdx.x; i0 < total; i0 += 8 * blockDim.x) {
        float x[8];
#pragma unroll
        for (int j = 0; j < 8; ++j) {
          const int i = i0 + j * blockDim.x;
          const int item = i / DP, c = i % DP, t = item >> 1, is_k = item & 1;
          x[j] = i < total && c < dim
                     ? to_f32<T>(qkv[static_cast<size_t>(q0 + t0 + t) * qkv_stride + (is_k ? k_col : q_col) + kvh * dim + c])
                     : 0.f;
        }
#pragma unroll
        for (int j = 0; j < 8; ++j) {
          const int i = i0 + j * blockDim.x;
          if (i < total) {
            const int item = i / DP, c = i % DP, t = item >> 1, is_k = item & 1;
            ((is_k ? ks : qs) + t * DS)[c] = is_k ? x[j] : x[j] * q_mul;
          }
        }
      }
    }
    if (per_channel) {
#pragma unroll 1
      for (int i = threadIdx.x; i < nt * DP; i += blockDim.x) {
        const int t = i / DP, c = i % DP;
        // (channels past dim decay to nothing: their rows of S are zeros anyway)
        as[t * DS + c] = c < dim ? channel_decay(decay[static_cast<size_t>(q0 + t0 + t) * decay_stride + decay_col + h * dim + c] + dec_bias[h * dim + c],
                                                 decay_mode, tau, dec_rate)
                                 : 0.f;
      }
    }
    for (int i = threadIdx.x; i < nt * cols_per_block; i += blockDim.x) {
      const int t = i / cols_per_block, c = col0 + i % cols_per_block;
      vs[i] = c < vdim ? to_f32<T>(qkv[static_cast<size_t>(q0 + t0 + t) * qkv_stride + v_col + h * vdim + c]) : 0.f;
    }
    for (int t = threadIdx.x; t < nt; t += blockDim.x) {
      const size_t n = static_cast<size_t>(q0 + t0 + t);
      const float step = decay_mode == 0 ? scan_softplus(decay[n * decay_stride + decay_col + h] + decay_p1[h]) : 1.f;
      if (decay_mode == 0) as[t] = expf(-expf(decay_p0[h]) * step);
      if (decay_mode == 4) as[t] = decay_p0[h];
      float b = write_mode == 2 ? step : 1.f;
      if (delta) b = 1.f / (1.f + expf(-(beta_rows != nullptr ? to_f32<T>(beta_rows[n * beta_stride + beta_col + h]) : beta[n * beta_stride + beta_col + h])));
      bs[t] = b;
    }
    __syncthreads();
    // eight lanes a token: unit norms (the rows scaled where they lie) and k . q, which the read-out needs;
    // the sums over a token's eight lanes are register exchanges
    for (int t = threadIdx.x / 8; t < nt; t += blockDim.x / 8) {
      const int s8 = threadIdx.x % 8;
      float* qrow = qs + t * DS;
      float* krow = ks + t * DS;
      float ssq = 0.f, ssk = 0.f, dot = 0.f;
      for (int c = 4 * s8; c < DP; c += 32) {
        const float4 a = *reinterpret_cast<const float4*>(qrow + c), b = *reinterpret_cast<const float4*>(krow + c);
        ssq = fmaf(a.x, a.x, fmaf(a.y, a.y, fmaf(a.z, a.z, fmaf(a.w, a.w, ssq))));
        ssk = fmaf(b.x, b.x, fmaf(b.y, b.y, fmaf(b.z, b.z, fmaf(b.w, b.w, ssk))));
        if (read_first) {
          const float4 u = *reinterpret_cast<const float4*>(us + c);
          dot = fmaf(a.x * u.x, b.x, fmaf(a.y * u.y, b.y, fmaf(a.z * u.z, b.z, fmaf(a.w * u.w, b.w, dot))));
        } else {
          dot = fmaf(a.x, b.x, fmaf(a.y, b.y, fmaf(a.z, b.z, fmaf(a.w, b.w, dot))));
        }
      }
      dot = column_sum<8>(dot);
      if (unit_eps >= 0.f) {
        const float mq = q_scale / sqrtf(column_sum<8>(ssq) + unit_eps), mk = 1.f / sqrtf(column_sum<8>(ssk) + unit_eps);
        for (int c = 4 * s8; c < DP; c += 32) {
          float4 a = *reinterpret_cast<const float4*>(qrow + c), b = *reinterpret_cast<const float4*>(krow + c);
          a.x *= mq; a.y *= mq; a.z *= mq; a.w *= mq;
          b.x *= mk; b.y *= mk; b.z *= mk; b.w *= mk;
          *reinterpret_cast<float4*>(qrow + c) = a;
          *reinterpret_cast<float4*>(krow + c) = b;
        }
        dot *= mq * mk;
      }
      if (s8 == 0) kqs[t] = dot;
    }
    __syncthreads();
    // the walk; a token's k, q and decays are read from LDS while the token before is worked on
    // (the token's scalars come with them: read where they are used, each costs the single wave of a SIMD a
    // round trip to LDS that nothing hides)
    float kn[kScanRows], qn[kScanRows], an[kScanRows];
    float a_n = 1.f, v_n = 0.f, b_n = 1.f, kq_n = 0.f;
    auto fetch = [&](int t) {
      if (!per_channel) a_n = as[t];
      v_n = vs[t * cols_per_block + col_local];
      b_n = bs[t];
      kq_n = kqs[t];
      const float4* kt = reinterpret_cast<const float4*>(ks + t * DS + sub * kScanRows);
      const float4* qt = reinterpret_cast<const float4*>(qs + t * DS + sub * kScanRows);
#pragma unroll
      for (int r4 = 0; r4 < kScanRows / 4; ++r4) {
        const float4 k4 = kt[r4], q4 = qt[r4];
        kn[4 * r4] = k4.x; kn[4 * r4 + 1] = k4.y; kn[4 * r4 + 2] = k4.z; kn[4 * r4 + 3] = k4.w;
        qn[4 * r4] = q4.x; qn[4 * r4 + 1] = q4.y; qn[4 * r4 + 2] = q4.z; qn[4 * r4 + 3] = q4.w;
      }
      if (per_channel) {
        const float4* at = reinterpret_cast<const float4*>(as + t * DS + sub * kScanRows);
#pragma unroll
        for (int r4 = 0; r4 < kScanRows / 4; ++r4) {
          const float4 a4 = at[r4];
          an[4 * r4] = a4.x; an[4 * r4 + 1] = a4.y; an[4 * r4 + 2] = a4.z; an[4 * r4 + 3] = a4.w;
        }
      }
    };
    fetch(0);
#pragma unroll 2
    for (int t = 0; t < nt; ++t) {
      float kr[kScanRows], qr[kScanRows];
#pragma unroll
      for (int r = 0; r < kScanRows; ++r) {
        kr[r] = kn[r];
        qr[r] = qn[r];
      }
      float pk[4] = {0.f, 0.f, 0.f, 0.f}, pq[4] = {0.f, 0.f, 0.f, 0.f};
      if (read_first) {
#pragma unroll
        for (int r = 0; r < kScanRows; ++r) pq[r % 4] = fmaf(S[r], qr[r], pq[r % 4]);
      }
      if (per_channel) {
#pragma unroll
        for (int r = 0; r < kScanRows; ++r) S[r] *= an[r];
      } else {
        const float a = a_n;
#pragma unroll
        for (int r = 0; r < kScanRows; ++r) S[r] *= a;
      }
      const float v_t = v_n, b_t = b_n, kq_t = kq_n;
      if (t + 1 < nt) fetch(t + 1);
      // both sums over the decayed S at once: S^T k for the write, S^T q for the read-out, which sees the
      // token's own write through q . (k u^T) = u (k . q)
      if (!read_first) {
#pragma unroll
        for (int r = 0; r < kScanRows; ++r) {
          pk[r % 4] = fmaf(S[r], kr[r], pk[r % 4]);
          pq[r % 4] = fmaf(S[r], qr[r], pq[r % 4]);
        }
      }
      const float sq = column_sum<TPC>((pq[0] + pq[1]) + (pq[2] + pq[3]));
      float u = v_t;
      if (delta) u = b_t * (u - column_sum<TPC>((pk[0] + pk[1]) + (pk[2] + pk[3])));
      else u *= b_t;  // (1 for plain writes)
      const float so = fmaf(skip_h, v_t, fmaf(u, kq_t, sq));
#pragma unroll
      for (int r = 0; r < kScanRows; ++r) S[r] = fmaf(kr[r], u, S[r]);
      if (has_col && sub == 0) out[(static_cast<size_t>(q0 + t0 + t) * n_heads + h) * vdim + col] = so;
    }
  }
#pragma unroll
  for (int r = 0; r < kScanRows; ++r) {
    const int i = sub * kScanRows + r;
    if (has_col && i < dim) S_head[static_cast<size_t>(i) * vdim + col] = S[r];
  }
}

// The form for aligned rows (what the engine's own tensors are).  Its loop over tokens is all that most of its time goes to, a
// wave alone on its SIMD with nothing to hide behind, so what a token costs in instructions is what counts: the kind of decay,
// write and read-out are template parameters (KIND, a sum of the flags below) and leave no branch in it; the next token's
// vectors are read from LDS into a second register set by turns, without moves; its scalars come as one 16-byte read.  The
// chunk after this one is on its way from memory while this one is walked.  Decays per channel are made by a kernel of
// their own first (GIVEN: `decay` holds them), or, for steps of few tokens, here while they are staged.
constexpr int kScanChannel = 1;    // a decay per key channel (else one for the head)
constexpr int kScanDelta = 2;      // the delta rule (else plain writes, or writes by the step)
constexpr int kScanReadFirst = 4;  // the read-out sees the memory as it was, plus the bonus

template <typename T>
struct Raw8;  // eight elements as they lie in memory
template <>
struct Raw8<bf16_t> {
  uint4 w;
  __device__ __forceinline__ void load(const bf16_t* p) { w = *reinterpret_cast<const uint4*>(p); }
  __device__ __forceinline__ void clear() { w = make_uint4(0u, 0u, 0u, 0u); }
  __device__ __forceinline__ void store(float* dst, float mul) const {
    *reinterpret_cast<float4*>(dst) = make_float4(__uint_as_float(w.x << 16) * mul, __uint_as_float(w.x & 0xffff0000u) * mul,
                                                  __uint_as_float(w.y << 16) * mul, __uint_as_float(w.y & 0xffff0000u) * mul);
    *reinterpret_cast<float4*>(dst + 4) = make_float4(__uint_as_float(w.z << 16) * mul, __uint_as_float(w.z & 0xffff0000u) * mul,
                                                      __uint_as_float(w.w << 16) * mul, __uint_as_float(w.w & 0xffff0000u) * mul);
  }
};
template <>
struct Raw8<float> {
  float4 a, b;
  __device__ __forceinline__ void load(const float* p) { a = *reinterpret_cast<const float4*>(p), b = *reinterpret_cast<const float4*>(p + 4); }
  __device__ __forceinline__ void clear() { a = b = make_float4(0.f, 0.f, 0.f, 0.f); }
  __device__ __forceinline__ void store(float* dst, float mul) const {
    *reinterpret_cast<float4*>(dst) = make_float4(a.x * mul, a.y * mul, a.z * mul, a.w * mul);
    *reinterpret_cast<float4*>(dst + 4) = make_float4(b.x * mul, b.y * mul, b.z * mul, b.w * mul);
  }
};

struct ScanArgs {
  const int32_t *seq_qstart, *seq_qlen, *state_slots;
  int qkv_stride, n_heads, n_kv, dim, vdim, q_col, k_col, v_col;
  float q_scale, unit_eps;
  int decay_mode, given;  // given: `decay` holds the channels' decays themselves
  const float* decay;
  int decay_stride, decay_col;
  const float *decay_p0, *decay_p1;
  float tau;
  const float* beta;
  int beta_stride, beta_col, by_step;
  const float *skip, *bonus;
  int chunk;
};

template <typename T, int TPC, int ROWS, int KIND>
__global__ __launch_bounds__(256) void linear_state_scan_fast_kernel(const T* __restrict__ qkv, float* __restrict__ state, float* __restrict__ out,
                                                                     const T* __restrict__ beta_rows, ScanArgs g) {
  constexpr bool CH = KIND & kScanChannel, DELTA = KIND & kScanDelta, FIRST = KIND & kScanReadFirst;
  constexpr int DP = TPC * ROWS;  // padded key channels
  constexpr int DS = DP + 4;      // a staged row's stride: rows of different tokens then start in different banks
  constexpr int COLS = 256 / TPC;
  constexpr int P8 = DP / 8, P4 = DP / 4;
  constexpr int NQ = DP / 32 < 1 ? 1 : (DP / 32 > 8 ? 8 : DP / 32);  // 16-byte pieces of q and k a thread stages (and of decays)
  constexpr int NV = kScanTokens / TPC < 1 ? 1 : kScanTokens / TPC;  // values a thread stages
  extern __shared__ float lds[];
  const int chunk = g.chunk, rows_staged = chunk + 2;  // (the walk reads up to two tokens ahead; what it finds there is not used)
  float* ks = lds;                                  // [chunk + 2][DS]
  float* qs = ks + rows_staged * DS;                // [chunk + 2][DS]
  float* as = qs + rows_staged * DS;                // [chunk + 2][DS] where decays are per channel
  float* sc = as + (CH ? rows_staged * DS : 0);     // [chunk + 2][4]: the head's decay, the write's strength, k . q (with the bonus)
  float* vs = sc + rows_staged * 4;                 // [chunk + 2][COLS]
  float* us = vs + rows_staged * COLS;              // [DP]: the head's bonus

  const int seq = blockIdx.x, h = blockIdx.y, kvh = h / (g.n_heads / g.n_kv);
  const int col0 = blockIdx.z * COLS;
  const int sub = threadIdx.x % TPC, col_local = threadIdx.x / TPC, col = col0 + col_local;
  const int dim = g.dim, vdim = g.vdim;
  const bool has_col = col < vdim;
  const int q0 = g.seq_qstart[seq], ql = g.seq_qlen[seq];
  float* S_head = state + (static_cast<size_t>(g.state_slots[seq]) * g.n_heads + h) * dim * vdim;
  const float skip_h = g.skip != nullptr ? g.skip[h] : 0.f;
  if (FIRST)
    for (int i = threadIdx.x; i < DP; i += 256) us[i] = i < dim ? g.bonus[h * dim + i] : 0.f;
  const float* dec_bias = g.decay_mode == 2 ? g.decay_p1 : g.decay_p0;
  const float dec_rate = CH && g.decay_mode == 2 && !g.given ? expf(g.decay_p0[h]) : 1.f;

  float S[ROWS];
#pragma unroll
  for (int r = 0; r < ROWS; ++r) {
    const int i = sub * ROWS + r;
    S[r] = has_col && i < dim ? S_head[static_cast<size_t>(i) * vdim + col] : 0.f;
  }

  // a chunk's operands, on their way in registers
  Raw8<T> qk[NQ];
  float4 dz[CH ? NQ : 1];
  T vv[NV];
  float s_dec = 0.f, s_beta = 0.f;
  auto ask = [&](int t0) {
    const int nt = min(chunk, ql - t0);
    const size_t n0 = static_cast<size_t>(q0 + t0);
#pragma unroll
    for (int j = 0; j < NQ; ++j) {
      const int v = threadIdx.x + j * 256;
      const int item = v / P8, c = 8 * (v % P8), t = item >> 1, is_k = item & 1;
      if (v < 2 * nt * P8 && c < dim)
        qk[j].load(qkv + (n0 + t) * g.qkv_stride + (is_k ? g.k_col : g.q_col) + kvh * dim + c);
      else
        qk[j].clear();
    }
    if (CH && g.given) {
#pragma unroll
      for (int j = 0; j < NQ; ++j) {
        const int v = threadIdx.x + j * 256, t = v / P4, c = 4 * (v % P4);
        // (channels past dim decay to nothing: their rows of S are zeros anyway)
        dz[CH ? j : 0] = v < nt * P4 && c < dim ? *reinterpret_cast<const float4*>(g.decay + (n0 + t) * g.decay_stride + g.decay_col + h * dim + c)
                                                : make_float4(0.f, 0.f, 0.f, 0.f);
      }
    }
#pragma unroll
    for (int j = 0; j < NV; ++j) {
      const int i = threadIdx.x + j * 256, t = i / COLS, c = col0 + i % COLS;
      vv[j] = i < nt * COLS && c < vdim ? qkv[(n0 + t) * g.qkv_stride + g.v_col + h * vdim + c] : T(0);
    }
    if (threadIdx.x < nt) {
      const size_t n = n0 + threadIdx.x;
      if (!CH && g.decay_mode == 0) s_dec = g.decay[n * g.decay_stride + g.decay_col + h];
      if (DELTA) s_beta = beta_rows != nullptr ? to_f32<T>(beta_rows[n * g.beta_stride + g.beta_col + h]) : g.beta[n * g.beta_stride + g.beta_col + h];
    }
  };

  ask(0);
  for (int t0 = 0; t0 < ql; t0 += chunk) {
    const int nt = min(chunk, ql - t0);
    __syncthreads();  // the chunk before has been read
    {
      const float q_mul = g.unit_eps >= 0.f ? 1.f : g.q_scale;
#pragma unroll
      for (int j = 0; j < NQ; ++j) {
        const int v = threadIdx.x + j * 256;
        const int item = v / P8, c = 8 * (v % P8), t = item >> 1, is_k = item & 1;
        if (v < 2 * nt * P8) qk[j].store((is_k ? ks : qs) + t * DS + c, is_k ? 1.f : q_mul);
      }
      if (CH && g.given) {
#pragma unroll
        for (int j = 0; j < NQ; ++j) {
          const int v = threadIdx.x + j * 256;
          if (v < nt * P4) *reinterpret_cast<float4*>(as + (v / P4) * DS + 4 * (v % P4)) = dz[CH ? j : 0];
        }
      }
#pragma unroll
      for (int j = 0; j < NV; ++j) {
        const int i = threadIdx.x + j * 256;
        if (i < nt * COLS) vs[i] = to_f32<T>(vv[j]);
      }
      if (threadIdx.x < nt) {
        const float step = CH || g.decay_mode != 0 ? 1.f : scan_softplus(s_dec + g.decay_p1[h]);
        if (!CH) sc[4 * threadIdx.x] = g.decay_mode == 4 ? g.decay_p0[h] : expf(-expf(g.decay_p0[h]) * step);
        sc[4 * threadIdx.x + 1] = DELTA ? 1.f / (1.f + expf(-s_beta)) : (g.by_step ? step : 1.f);
      }
      if (CH && !g.given) {
#pragma unroll 1
        for (int i = threadIdx.x; i < nt * DP; i += 256) {
          const int t = i / DP, c = i % DP;
          as[t * DS + c] = c < dim ? channel_decay(g.decay[static_cast<size_t>(q0 + t0 + t) * g.decay_stride + g.decay_col + h * dim + c] + dec_bias[h * dim + c],
                                                   g.decay_mode, g.tau, dec_rate)
                                   : 0.f;
        }
      }
    }
    __syncthreads();
    // eight lanes a token: unit norms (the rows scaled where they lie) and k . q, which the read-out needs
    for (int t = threadIdx.x / 8; t < nt; t += 32) {
      const int s8 = threadIdx.x % 8;
      float* qrow = qs + t * DS;
      float* krow = ks + t * DS;
      float ssq = 0.f, ssk = 0.f, dot = 0.f;
      for (int c = 4 * s8; c < DP; c += 32) {
        const float4 a = *reinterpret_cast<const float4*>(qrow + c), b = *reinterpret_cast<const float4*>(krow + c);
        ssq = fmaf(a.x, a.x, fmaf(a.y, a.y, fmaf(a.z, a.z, fmaf(a.w, a.w, ssq))));
        ssk = fmaf(b.x, b.x, fmaf(b.y, b.y, fmaf(b.z, b.z, fmaf(b.w, b.w, ssk))));
        if (FIRST) {
          const float4 u = *reinterpret_cast<const float4*>(us + c);
          dot = fmaf(a.x * u.x, b.x, fmaf(a.y * u.y, b.y, fmaf(a.z * u.z, b.z, fmaf(a.w * u.w, b.w, dot))));
        } else {
          dot = fmaf(a.x, b.x, fmaf(a.y, b.y, fmaf(a.z, b.z, fmaf(a.w, b.w, dot))));
        }
      }
      dot = column_sum<8>(dot);
      if (g.unit_eps >= 0.f) {
        const float mq = g.q_scale / sqrtf(column_sum<8>(ssq) + g.unit_eps), mk = 1.f / sqrtf(column_sum<8>(ssk) + g.unit_eps);
        for (int c = 4 * s8; c < DP; c += 32) {
          float4 a = *reinterpret_cast<const float4*>(qrow + c), b = *reinterpret_cast<const float4*>(krow + c);
          a.x *= mq; a.y *= mq; a.z *= mq; a.w *= mq;
          b.x *= mk; b.y *= mk; b.z *= mk; b.w *= mk;
          *reinterpret_cast<float4*>(qrow + c) = a;
          *reinterpret_cast<float4*>(krow + c) = b;
        }
        dot *= mq * mk;
      }
      if (s8 == 0) sc[4 * t + 2] = dot;
    }
    __syncthreads();
    if (t0 + chunk < ql) ask(t0 + chunk);
    // the walk: two register sets by turns
    struct Token {
      float4 k[ROWS / 4], q[ROWS / 4], a[CH ? ROWS / 4 : 1], s;
      float v;
    } one, two;
    const float *kp = ks + sub * ROWS, *qp = qs + sub * ROWS, *ap = as + sub * ROWS, *vp = vs + col_local, *sp = sc;
    auto fetch = [&](Token& x, int ahead) {
#pragma unroll
      for (int r = 0; r < ROWS / 4; ++r) {
        x.k[r] = *reinterpret_cast<const float4*>(kp + ahead * DS + 4 * r);
        x.q[r] = *reinterpret_cast<const float4*>(qp + ahead * DS + 4 * r);
        if (CH) x.a[r] = *reinterpret_cast<const float4*>(ap + ahead * DS + 4 * r);
      }
      x.s = *reinterpret_cast<const float4*>(sp + ahead * 4);
      x.v = vp[ahead * COLS];
    };
    float* op = out + (static_cast<size_t>(q0 + t0) * g.n_heads + h) * vdim + col;
    const size_t o_stride = static_cast<size_t>(g.n_heads) * vdim;
    const bool stores = has_col && sub == 0;
    auto walk = [&](const Token& x) {
      // both sums over S at once: S^T k for the write, S^T q for the read-out, which sees the token's own write through
      // q . (k u^T) = u (k . q)
      float pk[4] = {0.f, 0.f, 0.f, 0.f}, pq[4] = {0.f, 0.f, 0.f, 0.f};
      const float* k = reinterpret_cast<const float*>(x.k);
      const float* q = reinterpret_cast<const float*>(x.q);
      const float* a = reinterpret_cast<const float*>(x.a);
      if (FIRST) {
#pragma unroll
        for (int r = 0; r < ROWS; ++r) pq[r % 4] = fmaf(S[r], q[r], pq[r % 4]);
      }
#pragma unroll
      for (int r = 0; r < ROWS; ++r) S[r] *= CH ? a[CH ? r : 0] : x.s.x;
#pragma unroll
      for (int r = 0; r < ROWS; ++r) {
        if (DELTA) pk[r % 4] = fmaf(S[r], k[r], pk[r % 4]);
        if (!FIRST) pq[r % 4] = fmaf(S[r], q[r], pq[r % 4]);
      }
      float u = x.v;
      if (DELTA) u = x.s.y * (u - column_sum<TPC>((pk[0] + pk[1]) + (pk[2] + pk[3])));
      else if (!CH) u *= x.s.y;
      const float sq = column_sum<TPC>((pq[0] + pq[1]) + (pq[2] + pq[3]));
#pragma unroll
      for (int r = 0; r < ROWS; ++r) S[r] = fmaf(k[r], u, S[r]);
      float so = fmaf(u, x.s.z, sq);
      if (!CH && !DELTA) so = fmaf(skip_h, x.v, so);
      if (stores) *op = so;
      op += o_stride;
    };
    fetch(one, 0);
    int t = 0;
    for (; t + 1 < nt; t += 2) {
      fetch(two, 1);
      walk(one);
      fetch(one, 2);
      walk(two);
      kp += 2 * DS, qp += 2 * DS, ap += 2 * DS, vp += 2 * COLS, sp += 8;
    }
    if (t < nt) walk(one);
  }
#pragma unroll
  for (int r = 0; r < ROWS; ++r) {
    const int i = sub * ROWS + r;
    if (has_col && i < dim) S_head[static_cast<size_t>(i) * vdim + col] = S[r];
  }
}

// decays per key channel, made once for all the columns that will read them: out[n][h * dim + i], four a thread
__global__ __launch_bounds__(256) void channel_decay_kernel(const float* __restrict__ z, int stride, int col, const float* __restrict__ p0,
                                                            const float* __restrict__ p1, int mode, float tau, int dim, int channels,
                                                            float* __restrict__ out, size_t total4) {
  for (size_t i = blockIdx.x * static_cast<size_t>(blockDim.x) + threadIdx.x; i < total4; i += static_cast<size_t>(gridDim.x) * blockDim.x) {
    const size_t n = i / (channels / 4);
    const int c = 4 * static_cast<int>(i % (channels / 4));
    const float4 x = *reinterpret_cast<const float4*>(z + n * stride + col + c);
    const float4 b = *reinterpret_cast<const float4*>((mode == 2 ? p1 : p0) + c);
    const float rate = mode == 2 ? expf(p0[c / dim]) : 1.f;  // (a head's channels are a multiple of four)
    float v[4] = {x.x + b.x, x.y + b.y, x.z + b.z, x.w + b.w};
#pragma unroll 1
    for (int e = 0; e < 4; ++e) v[e] = channel_decay(v[e], mode, tau, rate);
    *reinterpret_cast<float4*>(out + n * channels + c) = make_float4(v[0], v[1], v[2], v[3]);
  }
}

// decay_mode 0: one decay per head from decay[n, decay_col + h], p0 = A_log [heads], p1 = dt_bias [heads];
// decay_mode 1, 2, 3: one per key channel from z = decay[n, decay_col + h * dim + i]: 1, sigmoid(z + p0)^(1 / tau), p0 =
// bias [heads * dim]; 2, exp(-exp(p0[h]) softplus(z + p1)), p0 = A_log [heads], p1 = dt_bias [heads * dim]; 3,
// exp(-exp(z + p0)), p0 = bias [heads * dim]; decay_mode 4: p0[h] itself, a constant per head (nothing is read per token).
// beta (float32) or, in its place, beta_rows (of qkv's dtype), both read at [n, beta_col + h].  bonus [heads * dim]
// float32 or null: the read-out comes before the write, with the token's own write weighed by the bonus (plain writes).
// decays [n_tokens][heads * dim] float32 or null: room for the decays per channel, made first where tokens are many.
// write_mode 0: plain writes; 1: the delta rule with beta = sigmoid(beta[n, beta_col + h]); 2: u = dt v with the
// step dt = softplus(decay[n, decay_col + h] + p1[h]) that the head's decay is made of (decay_mode 0 only).
// unit_eps < 0: q and k are taken as they are.  q_col, k_col, v_col: where the kv_heads' queries and keys and the
// heads' values start in a row of qkv.  skip [heads] or null: o += skip[h] v.
extern "C" int yk_linear_state_scan(const void* qkv, int qkv_stride, int dtype, int n_heads, int n_kv, int dim, int vdim,
                                    float* state, const int32_t* seq_qstart, const int32_t* seq_qlen,
                                    const int32_t* state_slots, int n_seqs, int n_tokens, float q_scale, float unit_eps, int decay_mode,
                                    const float* decay, int decay_stride, int decay_col, const float* decay_p0,
                                    const float* decay_p1, float tau, const float* beta, int beta_stride, int beta_col,
                                    float* out, int q_col, int k_col, int v_col, int write_mode, const float* skip,
                                    const void* beta_rows, const float* bonus, float* decays, hipStream_t stream) {
  YK_REQUIRE(n_seqs >= 0 && n_heads > 0 && n_kv > 0 && n_heads % n_kv == 0 && dim > 0 && vdim > 0, "linear_state_scan: bad sizes");
  YK_REQUIRE(q_col >= 0 && k_col >= 0 && v_col >= 0 && qkv_stride >= std::max(std::max(q_col, k_col) + n_kv * dim, v_col + n_heads * vdim),
             "linear_state_scan: rows shorter than q, k and v");
  YK_REQUIRE(write_mode == 0 || (write_mode == 1 && (beta != nullptr || beta_rows != nullptr)) || (write_mode == 2 && decay_mode == 0),
             "linear_state_scan: the delta rule needs beta, a write by the step the decay per head");
  YK_REQUIRE(decay_mode >= 0 && decay_mode <= 4, "linear_state_scan: unknown kind of decay");
  YK_REQUIRE(bonus == nullptr || (write_mode == 0 && skip == nullptr), "linear_state_scan: a bonus goes with plain writes and no skip");
  YK_REQUIRE(decay_p0 != nullptr && (decay_mode == 4 || (decay != nullptr && (decay_mode == 1 || decay_mode == 3 || decay_p1 != nullptr))), "linear_state_scan: the decay's inputs are missing");
  YK_REQUIRE(decay_mode != 1 || tau > 0.f, "linear_state_scan: tau must be positive");
  YK_REQUIRE(dim <= kScanRowsMax * kWave, "linear_state_scan: heads of more than 1,024 key channels are not offered");
  if (n_seqs == 0) return 0;
  const bool per_channel = decay_mode != 0 && decay_mode != 4;
  // eight rows a lane while that leaves a column inside a wave (a wave's instructions per token are what
  // the walk costs: fewer rows a lane, more lanes a column), sixteen beyond
  // (steps of single tokens are all staging and no walk: there the fewer, larger workgroups of sixteen rows
  // a lane stage less twice)
  const int rows = dim <= 8 * kWave && n_tokens > 4 * n_seqs ? 8 : 16;
  int tpc = 1;
  while (tpc * rows < dim) tpc *= 2;
  // (always 256 threads: columns a workgroup has no use for idle in the walk but help to stage)
  const int threads = 256;
  const int cols = threads / tpc;
  dim3 grid(n_seqs, n_heads, (vdim + cols - 1) / cols);
  const size_t dp = static_cast<size_t>(tpc) * rows;
  int chunk = kScanTokens;
  const size_t per_token = sizeof(float) * (2 * (dp + 4) + (per_channel ? dp + 4 : 1) + cols + 2);
  while (chunk > 4 && (chunk * per_token > 110 * 1024 || chunk * dp > 8192)) chunk /= 2;
  const size_t lds = chunk * per_token + (bonus != nullptr ? (dp + 4) * sizeof(float) : 0);
  YK_REQUIRE(lds <= 128 * 1024, "linear_state_scan: the staged tokens do not fit in LDS");
  auto al16 = [](const void* p) { return reinterpret_cast<uintptr_t>(p) % 16 == 0; };
  const int kind = (per_channel ? kScanChannel : 0) + (write_mode == 1 ? kScanDelta : 0) + (bonus != nullptr ? kScanReadFirst : 0);
  const bool fast = dim % 8 == 0 && qkv_stride % 8 == 0 && q_col % 8 == 0 && k_col % 8 == 0 && al16(qkv) && chunk * dp <= 8192 && kind != kScanReadFirst &&
                    (skip == nullptr || kind == 0);
  if (fast) {
    // many tokens: their decays per channel first, where the caller gave room for them
    const bool given = per_channel && decays != nullptr && decay_stride % 4 == 0 && decay_col % 4 == 0 && al16(decay) && al16(decays) &&
                       al16(decay_mode == 2 ? decay_p1 : decay_p0);
    if (given) {
      const size_t total4 = static_cast<size_t>(n_tokens) * n_heads * dim / 4;
      const int dgrid = static_cast<int>(std::min<size_t>((total4 + 255) / 256, 1 << 20));
      channel_decay_kernel<<<dgrid, 256, 0, stream>>>(decay, decay_stride, decay_col, decay_p0, decay_p1, decay_mode, tau, dim, n_heads * dim, decays, total4);
      if (yk_check_launch("channel_decay")) return -1;
    }
    const ScanArgs g{seq_qstart, seq_qlen, state_slots, qkv_stride, n_heads, n_kv, dim, vdim, q_col, k_col, v_col, q_scale, unit_eps,
                     decay_mode, given, given ? decays : decay, given ? n_heads * dim : decay_stride, given ? 0 : decay_col, decay_p0, decay_p1, tau,
                     beta, beta_stride, beta_col, write_mode == 2, skip, bonus, chunk};
    const size_t fast_lds = sizeof(float) * ((chunk + 2) * ((per_channel ? 3 : 2) * (dp + 4) + 4 + cols) + dp);
    YK_REQUIRE(fast_lds <= 128 * 1024, "linear_state_scan: the staged tokens do not fit in LDS");
#define YK_FAST(T, TPC, KIND)                                                                                                   \
  {                                                                                                                             \
    auto kern = rows == 8 ? linear_state_scan_fast_kernel<T, TPC, 8, KIND> : linear_state_scan_fast_kernel<T, TPC, 16, KIND>;   \
    if (fast_lds > 64 * 1024 && hipFuncSetAttribute(reinterpret_cast<const void*>(kern), hipFuncAttributeMaxDynamicSharedMemorySize, \
                                                    static_cast<int>(fast_lds)) != hipSuccess)                                  \
      return yk_fail("linear_state_scan: the staged tokens do not fit in LDS");                                                 \
    kern<<<grid, threads, fast_lds, stream>>>(static_cast<const T*>(qkv), state, out, static_cast<const T*>(beta_rows), g);     \
    return yk_check_launch("linear_state_scan");                                                                                \
  }
#define YK_FAST_KIND(T, TPC)             \
  switch (kind) {                        \
    case 0: YK_FAST(T, TPC, 0)           \
    case 1: YK_FAST(T, TPC, 1)           \
    case 2: YK_FAST(T, TPC, 2)           \
    case 3: YK_FAST(T, TPC, 3)           \
    default: YK_FAST(T, TPC, 5)          \
  }
#define YK_FAST_TPC(T)                   \
  switch (tpc) {                         \
    case 1: YK_FAST_KIND(T, 1)           \
    case 2: YK_FAST_KIND(T, 2)           \
    case 4: YK_FAST_KIND(T, 4)           \
    case 8: YK_FAST_KIND(T, 8)           \
    case 16: YK_FAST_KIND(T, 16)         \
    case 32: YK_FAST_KIND(T, 32)         \
    default: YK_FAST_KIND(T, 64)         \
  }
    if (dtype == YK_F32) YK_FAST_TPC(float)
    if (dtype == YK_BF16) YK_FAST_TPC(bf16_t)
#undef YK_FAST_TPC
#undef YK_FAST_KIND
#undef YK_FAST
    return yk_fail("linear_state_scan: unsupported dtype");
  }
#define YK_LAUNCH(T, TPC)                                                                                                       \
  {                                                                                                                             \
    auto kern = rows == 8 ? linear_state_scan_kernel<T, TPC, 8> : linear_state_scan_kernel<T, TPC, 16>;                         \
    if (lds > 64 * 1024 && hipFuncSetAttribute(reinterpret_cast<const void*>(kern), hipFuncAttributeMaxDynamicSharedMemorySize, \
                                               static_cast<int>(lds)) != hipSuccess)                                            \
      return yk_fail("linear_state_scan: the staged tokens do not fit in LDS");                                                 \
    kern<<<grid, threads, lds, stream>>>(static_cast<const T*>(qkv), qkv_stride, n_heads, n_kv, dim, vdim, state, seq_qstart,   \
                                         seq_qlen, state_slots, q_scale, unit_eps, decay_mode, decay, decay_stride, decay_col,  \
                                         decay_p0, decay_p1, tau, beta, beta_stride, beta_col, chunk, out, q_col, k_col,       \
                                         v_col, write_mode, skip, static_cast<const T*>(beta_rows), bonus);                     \
    return yk_check_launch("linear_state_scan");                                                                                \
  }
#define YK_TPC(T)                   \
  switch (tpc) {                    \
    case 1: YK_LAUNCH(T, 1)         \
    case 2: YK_LAUNCH(T, 2)         \
    case 4: YK_LAUNCH(T, 4)         \
    case 8: YK_LAUNCH(T, 8)         \
    case 16: YK_LAUNCH(T, 16)       \
    case 32: YK_LAUNCH(T, 32)       \
    default: YK_LAUNCH(T, 64)       \
  }
  if (dtype == YK_F32) YK_TPC(float)
  if (dtype == YK_BF16) YK_TPC(bf16_t)
#undef YK_TPC
#undef YK_LAUNCH
  return yk_fail("linear_state_scan: unsupported dtype");
}

// ------------------------------------------------------------------------ what enters a recurrence
// float32 rows [q | k | v] from a projection's rows [q | k | v | ...]: with silu, the activation of all three; with tables,
// q and k rotated by their positions (the first `rot` elements of every head); k times k_scale.  A thread an element.
template <typename T>
__global__ __launch_bounds__(256) void scan_inputs_kernel(const T* __restrict__ src, int src_stride, int n_heads, int dim, int vdim,
                                                          const int32_t* __restrict__ positions, const float* __restrict__ cos_t,
                                                          const float* __restrict__ sin_t, int rot, int interleaved, int max_pos,
                                                          float k_scale, int silu, float* __restrict__ out, size_t total) {
  const int kd = n_heads * dim, cols = 2 * kd + n_heads * vdim;
  for (size_t i = blockIdx.x * static_cast<size_t>(blockDim.x) + threadIdx.x; i < total; i += static_cast<size_t>(gridDim.x) * blockDim.x) {
    const size_t n = i / cols;
    const int c = static_cast<int>(i % cols);
    const T* row = src + n * src_stride;
    auto at = [&](int col) { const float x = to_f32<T>(row[col]); return silu ? act_silu(x) : x; };
    float v = at(c);
    if (c < 2 * kd) {
      const int d = c % dim;
      if (d < rot) {
        const int half = rot / 2, m = interleaved ? d / 2 : (d < half ? d : d - half);
        const size_t a = static_cast<size_t>(min(positions[n], max_pos - 1)) * half + m;
        const bool first = interleaved ? d % 2 == 0 : d < half;
        const float other = at(interleaved ? (first ? c + 1 : c - 1) : (first ? c + half : c - half));
        v = first ? rot_first(v, other, cos_t[a], sin_t[a]) : rot_second(other, v, cos_t[a], sin_t[a]);
      }
      if (c >= kd) v *= k_scale;
    }
    out[i] = v;
  }
}

extern "C" int yk_scan_inputs(const void* src, int src_stride, int dtype, int n_heads, int dim, int vdim, const int32_t* positions,
                              const float* cos_t, const float* sin_t, int rot, int interleaved, int max_pos, float k_scale, int silu,
                              float* out, int n_tokens, hipStream_t stream) {
  YK_REQUIRE(n_tokens >= 0 && n_heads > 0 && dim > 0 && vdim > 0 && src_stride >= n_heads * (2 * dim + vdim), "scan_inputs: bad sizes");
  YK_REQUIRE(rot >= 0 && rot % 2 == 0 && rot <= dim && (rot == 0 || (cos_t != nullptr && sin_t != nullptr && positions != nullptr && max_pos > 0)),
             "scan_inputs: rotary tables missing, or more elements than a head has");
  if (n_tokens == 0) return 0;
  const size_t total = static_cast<size_t>(n_tokens) * n_heads * (2 * dim + vdim);
  const int grid = static_cast<int>(std::min<size_t>((total + 255) / 256, 1 << 20));
  if (dtype == YK_F32)
    scan_inputs_kernel<float><<<grid, 256, 0, stream>>>(static_cast<const float*>(src), src_stride, n_heads, dim, vdim, positions, cos_t, sin_t, rot,
                                                        interleaved, max_pos, k_scale, silu, out, total);
  else if (dtype == YK_BF16)
    scan_inputs_kernel<bf16_t><<<grid, 256, 0, stream>>>(static_cast<const bf16_t*>(src), src_stride, n_heads, dim, vdim, positions, cos_t, sin_t, rot,
                                                         interleaved, max_pos, k_scale, silu, out, total);
  else
    return yk_fail("scan_inputs: unsupported dtype");
  return yk_check_launch("scan_inputs");
}

// --------------------------------------------------------------- the read-out's norm and gate
// a wave per (token, part of vdim elements): y = o / sqrt(mean(o^2) + eps) * w * silu(gate), or, gate_first, the gate
// before the norm: y = g / sqrt(mean(g^2) + eps) * w with g = o * silu(gate).  gate_act 1: the sigmoid in silu's place.  w_stride 0: one weight of vdim elements
// for every part; vdim: a weight of n_heads * vdim elements; w null: no weight.
__device__ __forceinline__ float head_gate_act(float g, int act) { return act == 1 ? 1.f / (1.f + expf(-g)) : act_silu(g); }
template <typename TW, typename TG, typename TO>
__global__ __launch_bounds__(256) void gated_head_norm_kernel(const float* __restrict__ o, const TW* __restrict__ w, float eps,
                                                              const TG* __restrict__ gate, int gate_stride, int gate_col,
                                                              int n_heads, int vdim, TO* __restrict__ out, size_t total,
                                                              int w_stride, int gate_first, int gate_act) {
  const size_t item = blockIdx.x * static_cast<size_t>(blockDim.x / kWave) + threadIdx.x / kWave;
  if (item >= total) return;
  const int lane = threadIdx.x % kWave;
  const size_t n = item / n_heads;
  const int h = static_cast<int>(item % n_heads);
  const float* row = o + item * vdim;
  const TG* g = gate + n * gate_stride + gate_col + h * vdim;
  const TW* wp = w != nullptr ? w + static_cast<size_t>(h) * w_stride : nullptr;
  auto weight = [&](int c) { return wp != nullptr ? to_f32<TW>(wp[c]) : 1.f; };
  float ss = 0.f;
  if (gate_first) {
    for (int c = lane; c < vdim; c += kWave) {
      const float v = row[c] * head_gate_act(to_f32<TG>(g[c]), gate_act);
      ss = fmaf(v, v, ss);
    }
    const float inv = 1.f / sqrtf(wave_sum(ss) / static_cast<float>(vdim) + eps);
    for (int c = lane; c < vdim; c += kWave)
      out[item * vdim + c] = from_f32<TO>(row[c] * head_gate_act(to_f32<TG>(g[c]), gate_act) * inv * weight(c));
    return;
  }
  for (int c = lane; c < vdim; c += kWave) ss = fmaf(row[c], row[c], ss);
  const float inv = 1.f / sqrtf(wave_sum(ss) / static_cast<float>(vdim) + eps);
  for (int c = lane; c < vdim; c += kWave)
    out[item * vdim + c] = from_f32<TO>(row[c] * inv * weight(c) * head_gate_act(to_f32<TG>(g[c]), gate_act));
}

// The same in pieces of four elements, a thread holding up to four of them: everything is asked for before the sum.  A wave a
// part (four parts a workgroup) or, for parts of more than 1,024 elements, a workgroup a part.
template <typename T>
__device__ __forceinline__ float4 hn_load4(const T* p);
template <>
__device__ __forceinline__ float4 hn_load4<float>(const float* p) { return *reinterpret_cast<const float4*>(p); }
template <>
__device__ __forceinline__ float4 hn_load4<bf16_t>(const bf16_t* p) {
  const uint2 w = *reinterpret_cast<const uint2*>(p);
  return make_float4(__uint_as_float(w.x << 16), __uint_as_float(w.x & 0xffff0000u), __uint_as_float(w.y << 16), __uint_as_float(w.y & 0xffff0000u));
}
__device__ __forceinline__ void hn_store4(float* p, float4 v) { *reinterpret_cast<float4*>(p) = v; }
__device__ __forceinline__ void hn_store4(bf16_t* p, float4 v) { *reinterpret_cast<uint2*>(p) = make_uint2(pack_bf16x2(v.x, v.y), pack_bf16x2(v.z, v.w)); }

template <typename TW, typename TG, typename TO, bool WAVE>
__global__ __launch_bounds__(256) void gated_head_norm_vec_kernel(const float* __restrict__ o, const TW* __restrict__ w, float eps,
                                                                  const TG* __restrict__ gate, int gate_stride, int gate_col, int n_heads,
                                                                  int vdim, TO* __restrict__ out, size_t total, int w_stride, int gate_first,
                                                                  int gate_act) {
  __shared__ float scratch[17];
  constexpr int T = WAVE ? kWave : 256, P = 4;
  const size_t wanted = WAVE ? blockIdx.x * static_cast<size_t>(4) + threadIdx.x / kWave : blockIdx.x;
  if (WAVE && wanted >= total) return;  // (a whole wave)
  const size_t item = wanted;
  const int t = threadIdx.x % T;
  const size_t n = item / n_heads;
  const int h = static_cast<int>(item % n_heads);
  const float* row = o + item * vdim;
  const TG* g = gate + n * gate_stride + gate_col + h * vdim;
  float4 v[P], a[P], m[P];
  float ss = 0.f;
#pragma unroll
  for (int p = 0; p < P; ++p) {
    const int c = 4 * (t + p * T);
    v[p] = a[p] = make_float4(0.f, 0.f, 0.f, 0.f);
    m[p] = make_float4(1.f, 1.f, 1.f, 1.f);
    if (c < vdim) {
      v[p] = hn_load4<float>(row + c);
      a[p] = hn_load4<TG>(g + c);
      if (w != nullptr) m[p] = hn_load4<TW>(w + static_cast<size_t>(h) * w_stride + c);
    }
  }
#pragma unroll
  for (int p = 0; p < P; ++p) {
    a[p] = make_float4(head_gate_act(a[p].x, gate_act), head_gate_act(a[p].y, gate_act), head_gate_act(a[p].z, gate_act), head_gate_act(a[p].w, gate_act));
    if (gate_first) v[p] = make_float4(v[p].x * a[p].x, v[p].y * a[p].y, v[p].z * a[p].z, v[p].w * a[p].w);
    ss = fmaf(v[p].x, v[p].x, fmaf(v[p].y, v[p].y, fmaf(v[p].z, v[p].z, fmaf(v[p].w, v[p].w, ss))));
  }
  ss = WAVE ? wave_sum(ss) : block_sum(ss, scratch);
  const float inv = 1.f / sqrtf(ss / static_cast<float>(vdim) + eps);
#pragma unroll
  for (int p = 0; p < P; ++p) {
    const int c = 4 * (t + p * T);
    if (c < vdim) {
      float4 y = make_float4(v[p].x * inv * m[p].x, v[p].y * inv * m[p].y, v[p].z * inv * m[p].z, v[p].w * inv * m[p].w);
      if (!gate_first) y.x *= a[p].x, y.y *= a[p].y, y.z *= a[p].z, y.w *= a[p].w;
      hn_store4(out + item * vdim + c, y);
    }
  }
}

extern "C" int yk_gated_head_norm(const float* o, const void* w, int w_dtype, float eps, const void* gate, int gate_dtype,
                                  int gate_stride, int gate_col, int n_heads, int vdim, void* out, int out_dtype, int n_tokens,
                                  int w_per_part, int gate_first, int gate_act, hipStream_t stream) {
  YK_REQUIRE(n_tokens >= 0 && n_heads > 0 && vdim > 0 && gate_stride >= gate_col + n_heads * vdim, "gated_head_norm: bad sizes");
  YK_REQUIRE(gate_dtype == out_dtype || gate_dtype == YK_F32, "gated_head_norm: the gate comes in the output's dtype or float32");
  YK_REQUIRE(gate_act == 0 || gate_act == 1, "gated_head_norm: the gate is silu or the sigmoid");
  if (n_tokens == 0) return 0;
  const size_t total = static_cast<size_t>(n_tokens) * n_heads;
  const int grid = static_cast<int>((total + 3) / 4);
  const int w_stride = w_per_part ? vdim : 0;
  auto al16 = [](const void* p) { return reinterpret_cast<uintptr_t>(p) % 16 == 0; };
  const bool vec = vdim % 4 == 0 && vdim <= 4096 && gate_stride % 4 == 0 && gate_col % 4 == 0 && al16(o) && al16(w) && al16(gate) && al16(out);
#define YK_CASE(WD, TW, GD, TG, OD, TO)                                                                               \
  if (w_dtype == WD && gate_dtype == GD && out_dtype == OD) {                                                         \
    if (vec && vdim > 1024)                                                                                           \
      gated_head_norm_vec_kernel<TW, TG, TO, false><<<static_cast<unsigned>(total), 256, 0, stream>>>(                \
          o, static_cast<const TW*>(w), eps, static_cast<const TG*>(gate), gate_stride, gate_col, n_heads, vdim,      \
          static_cast<TO*>(out), total, w_stride, gate_first, gate_act);                                              \
    else if (vec)                                                                                                     \
      gated_head_norm_vec_kernel<TW, TG, TO, true><<<grid, 256, 0, stream>>>(                                         \
          o, static_cast<const TW*>(w), eps, static_cast<const TG*>(gate), gate_stride, gate_col, n_heads, vdim,      \
          static_cast<TO*>(out), total, w_stride, gate_first, gate_act);                                              \
    else                                                                                                              \
    gated_head_norm_kernel<TW, TG, TO><<<grid, 256, 0, stream>>>(o, static_cast<const TW*>(w), eps,                   \
                                                                 static_cast<const TG*>(gate), gate_stride, gate_col, \
                                                                 n_heads, vdim, static_cast<TO*>(out), total, w_stride, \
                                                                 gate_first, gate_act);                               \
    return yk_check_launch("gated_head_norm");                                                                        \
  }
  YK_CASE(YK_F32, float, YK_F32, float, YK_F32, float)
  YK_CASE(YK_BF16, bf16_t, YK_BF16, bf16_t, YK_BF16, bf16_t)
  YK_CASE(YK_F32, float, YK_BF16, bf16_t, YK_BF16, bf16_t)
  YK_CASE(YK_BF16, bf16_t, YK_F32, float, YK_BF16, bf16_t)
  YK_CASE(YK_F32, float, YK_F32, float, YK_BF16, bf16_t)
#undef YK_CASE
  return yk_fail("gated_head_norm: unsupported dtype combination");
}

// ------------------------------------------------------------ a convolution's kept inputs
// state [slots][keep][channels] holds a request's last `keep` inputs, oldest first; after a span of
// ql tokens it holds the last `keep` of (old state, the span's inputs).  A thread per (request, channel).
template <typename T>
__global__ void conv_state_push_kernel(const T* __restrict__ x, int x_stride, T* __restrict__ state,
                                       const int32_t* __restrict__ seq_qstart, const int32_t* __restrict__ seq_qlen,
                                       const int32_t* __restrict__ state_slots, int keep, int channels, size_t total) {
  for (size_t i = blockIdx.x * static_cast<size_t>(blockDim.x) + threadIdx.x; i < total;
       i += static_cast<size_t>(gridDim.x) * blockDim.x) {
    const int seq = static_cast<int>(i / channels), c = static_cast<int>(i % channels);
    const int q0 = seq_qstart[seq], ql = seq_qlen[seq];
    T* st = state + static_cast<size_t>(state_slots[seq]) * keep * channels + c;
    // new[j] = old[j + ql] while that exists, else the span's input ql - keep + j; ascending j reads
    // old rows before they are overwritten (j + ql > j)
    for (int j = 0; j < keep; ++j) {
      const int from = j + ql;
      st[static_cast<size_t>(j) * channels] =
          from < keep ? st[static_cast<size_t>(from) * channels] : x[static_cast<size_t>(q0 + from - keep) * x_stride + c];
    }
  }
}

extern "C" int yk_conv_state_push(const void* x, int x_stride, int dtype, void* state, const int32_t* seq_qstart,
                                  const int32_t* seq_qlen, const int32_t* state_slots, int n_seqs, int keep, int channels,
                                  hipStream_t stream) {
  YK_REQUIRE(n_seqs >= 0 && keep >= 0 && channels > 0 && x_stride >= channels, "conv_state_push: bad sizes");
  if (n_seqs == 0 || keep == 0) return 0;
  const size_t total = static_cast<size_t>(n_seqs) * channels;
  const int grid = static_cast<int>(std::min<size_t>((total + 255) / 256, 1 << 20));
  if (dtype == YK_F32)
    conv_state_push_kernel<float><<<grid, 256, 0, stream>>>(static_cast<const float*>(x), x_stride, static_cast<float*>(state),
                                                            seq_qstart, seq_qlen, state_slots, keep, channels, total);
  else if (dtype == YK_BF16)
    conv_state_push_kernel<bf16_t><<<grid, 256, 0, stream>>>(static_cast<const bf16_t*>(x), x_stride, static_cast<bf16_t*>(state),
                                                             seq_qstart, seq_qlen, state_slots, keep, channels, total);
  else
    return yk_fail("conv_state_push: unsupported dtype");
  return yk_check_launch("conv_state_push");
}
