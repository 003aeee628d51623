// The recurrence with a constant decay per head, S [dim][vdim] float32 in the request's state slot:
//
//   S <- a_h S + k_t v_t^T,   o_t = S^T q_t
//
// on a projection's rows [q | k | v | ...], of which q and k are rotated by their positions and k is scaled, or all three pass silu,
// in float32 on their way in (the plain form of the same is yk_scan_inputs and then yk_linear_state_scan with fixed decays).
//
// Because a decay is a power of a constant, the tokens of a chunk (up to 64) meet in matrix products.  With i, j the places
// in a chunk of n tokens and S the memory before it:
//
//   o_i   = a^(i+1) S^T q_i + sum over j <= i of a^(i-j) (q_i . k_j) v_j
//   S_end = a^n S + sum over j of a^(n-1-j) k_j v_j^T
//
// yk_decay_scan_chunks runs four kernels over a step's chunks (of all its requests):
//   * prepare: q, k (rows of the chunk), the weighed keys a^(n-1-j) k_j and the values (both transposed: a row of 64 tokens per
//     channel), everything rotated / activated once;
//   * inside: W_c = (sum of weighed k_j v_j^T)^T per chunk and head, on the matrix cores;
//   * across: per request, head and element, S = a^n S + W_c along its chunks; what stood before each chunk is left in W_c's place;
//   * out: both terms of o on the matrix cores.
// Operands of the matrix cores are bfloat16, so every float32 number goes in as two, x = hi + lo (16 bits of fraction): a
// product of two such is hi hi + hi lo + lo hi, summed in float32.  Eight numbers lie together as [8 hi | 8 lo], 32 bytes, so that
// a lane's two operand pieces are neighbours; a chunk's sum in float32 and the memory in two parts then take the same 32
// bytes, and the one replaces the other in place.  Values that are bfloat16 already (no activation) have no lo.
//
// yk_decay_scan_step is the step of single tokens: a workgroup per (request, head, 64 columns), every thread four neighbouring columns
// of every 16th row, the rows asked for before q, k and v are made.
#include <algorithm>

#include "common.h"

namespace {

typedef __bf16 bf16x8_t __attribute__((ext_vector_type(8)));
typedef float f32x4_t __attribute__((ext_vector_type(4)));
typedef uint32_t u32x4_t __attribute__((ext_vector_type(4)));
union Frag {
  u32x4_t u;
  bf16x8_t v;
};
struct Pair {
  Frag hi, lo;
};

constexpr int kChunk = 64;

// how q and k become what enters the recurrence
struct Inputs {
  const int32_t* positions;
  const float *cos_t, *sin_t;
  int rot, interleaved, max_pos;
  float k_scale;
  int silu;
};

template <typename T>
__device__ __forceinline__ void load8(const T* p, float* out);
template <>
__device__ __forceinline__ void load8<bf16_t>(const bf16_t* p, float* out) {
  const uint4 w = *reinterpret_cast<const uint4*>(p);
  out[0] = __uint_as_float(w.x << 16); out[1] = __uint_as_float(w.x & 0xffff0000u);
  out[2] = __uint_as_float(w.y << 16); out[3] = __uint_as_float(w.y & 0xffff0000u);
  out[4] = __uint_as_float(w.z << 16); out[5] = __uint_as_float(w.z & 0xffff0000u);
  out[6] = __uint_as_float(w.w << 16); out[7] = __uint_as_float(w.w & 0xffff0000u);
}

// eight floats as [8 hi | 8 lo] (dst in units of 8 numbers = 16 elements), or as 8 hi alone
__device__ __forceinline__ void split8(const float* v, u32x4_t& hi, u32x4_t& lo) {
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const uint32_t h = pack_bf16x2(v[2 * i], v[2 * i + 1]);
    hi[i] = h;
    lo[i] = pack_bf16x2(v[2 * i] - __uint_as_float(h << 16), v[2 * i + 1] - __uint_as_float(h & 0xffff0000u));
  }
}
__device__ __forceinline__ void store_pair(bf16_t* dst, const float* v) {
  u32x4_t hi, lo;
  split8(v, hi, lo);
  *reinterpret_cast<u32x4_t*>(dst) = hi;
  *reinterpret_cast<u32x4_t*>(dst + 8) = lo;
}
__device__ __forceinline__ Pair load_pair(const bf16_t* p) {
  Pair x;
  x.hi.u = *reinterpret_cast<const u32x4_t*>(p);
  x.lo.u = *reinterpret_cast<const u32x4_t*>(p + 8);
  return x;
}
__device__ __forceinline__ f32x4_t mma(const Frag& a, const Frag& b, f32x4_t c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a.v, b.v, c, 0, 0, 0);
}
__device__ __forceinline__ f32x4_t mma_pairs(const Pair& a, const Pair& b, f32x4_t c) {
  return mma(a.lo, b.hi, mma(a.hi, b.lo, mma(a.hi, b.hi, c)));
}

// elements 8p .. 8p + 7 of a head's q or k (row: where the head starts), rotated by position pos or through silu, times mul
__device__ __forceinline__ void enter8(const bf16_t* row, int p, int pos, const Inputs& in, float mul, float* v) {
  load8<bf16_t>(row + 8 * p, v);
  if (in.silu) {
#pragma unroll
    for (int e = 0; e < 8; ++e) v[e] = act_silu(v[e]);
  }
  if (8 * p < in.rot) {
    const int half = in.rot / 2;
    const size_t at = static_cast<size_t>(min(pos, in.max_pos - 1)) * half;
    if (in.interleaved) {
#pragma unroll
      for (int e = 0; e < 8; e += 2) {
        const float c = in.cos_t[at + 4 * p + e / 2], s = in.sin_t[at + 4 * p + e / 2], a = v[e], b = v[e + 1];
        v[e] = rot_first(a, b, c, s);
        v[e + 1] = rot_second(a, b, c, s);
      }
    } else {
      const bool first = 8 * p < half;
      const int m = 8 * p - (first ? 0 : half);
      float w[8];
      load8<bf16_t>(row + (first ? 8 * p + half : 8 * p - half), w);
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        const float c = in.cos_t[at + m + e], s = in.sin_t[at + m + e];
        v[e] = first ? rot_first(v[e], w[e], c, s) : rot_second(w[e], v[e], c, s);
      }
    }
  }
#pragma unroll
  for (int e = 0; e < 8; ++e) v[e] *= mul;
}

}  // namespace

// ---------------------------------------------------------------------------------------- chunks: prepare
// A workgroup a (chunk, head, block of 64 channels of q, of k or of v).  q_ws, k_ws [chunk][head][64][dim], kt_ws
// [chunk][head][dim][64], pairs of 8; vt_ws [chunk][head][vdim][64], pairs of 8 or (VLO false) hi alone.  Places beyond the
// chunk's tokens are zeros.
constexpr int kPrepare = 64;  // channels of a workgroup
template <bool VLO>
__global__ __launch_bounds__(256) void decay_prepare_kernel(const bf16_t* __restrict__ src, int src_stride, int n_heads, int dim, int vdim,
                                                            const float* __restrict__ decay, const int32_t* __restrict__ chunks, Inputs in,
                                                            bf16_t* __restrict__ q_ws, bf16_t* __restrict__ k_ws, bf16_t* __restrict__ kt_ws,
                                                            bf16_t* __restrict__ vt_ws) {
  __shared__ float buf[kChunk][kPrepare + 1];
  __shared__ float power[kChunk];
  const int c = blockIdx.x, h = blockIdx.y;
  const int tok0 = chunks[3 * c + 1], n = chunks[3 * c + 2];
  const size_t slab = static_cast<size_t>(c) * n_heads + h;
  const int key_blocks = (dim + kPrepare - 1) / kPrepare;
  const int what = min(static_cast<int>(blockIdx.z) / key_blocks, 2);  // 0: q, 1: k, 2: v
  const int c0 = (blockIdx.z - what * key_blocks) * kPrepare;            // its first channel
  const int width = what == 2 ? vdim : dim, here = min(kPrepare, width - c0), pieces = here / 8;
  const bf16_t* col = src + (what == 2 ? 2 * n_heads * dim + h * vdim : what * n_heads * dim + h * dim);
  if (what == 1 && threadIdx.x < kChunk) power[threadIdx.x] = powf(decay[h], static_cast<float>(threadIdx.x));
  for (int i = threadIdx.x; i < kChunk * pieces; i += 256) {
    const int t = i / pieces, p = c0 / 8 + i % pieces;
    float v[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
    if (t < n) {
      const bf16_t* row = col + static_cast<size_t>(tok0 + t) * src_stride;
      if (what == 2) {
        load8<bf16_t>(row + 8 * p, v);
        if (VLO) {
#pragma unroll
          for (int e = 0; e < 8; ++e) v[e] = act_silu(v[e]);
        }
      } else {
        enter8(row, p, in.positions[tok0 + t], in, what == 1 ? in.k_scale : 1.f, v);
      }
    }
    if (what != 2) store_pair((what == 0 ? q_ws : k_ws) + ((slab * kChunk + t) * (dim / 8) + p) * 16, v);
    if (what != 0) {
#pragma unroll
      for (int e = 0; e < 8; ++e) buf[t][8 * p - c0 + e] = v[e];
    }
  }
  if (what == 0) return;
  __syncthreads();
  // transposed: lanes side by side over a channel's pieces of eight tokens, so that a channel's row is written whole
  for (int i = threadIdx.x; i < here * (kChunk / 8); i += 256) {
    const int d = i / (kChunk / 8), p = i % (kChunk / 8);
    float v[8];
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      const int t = 8 * p + e;
      v[e] = what == 2 ? buf[t][d] : (t < n ? buf[t][d] * power[n - 1 - t] : 0.f);
    }
    const size_t at = (slab * width + c0 + d) * (kChunk / 8) + p;
    if (what == 1) {
      store_pair(kt_ws + at * 16, v);
    } else if (VLO) {
      store_pair(vt_ws + at * 16, v);
    } else {
      u32x4_t hi, lo;
      split8(v, hi, lo);
      *reinterpret_cast<u32x4_t*>(vt_ws + at * 8) = hi;
    }
  }
}

// ---------------------------------------------------------------------------------------- chunks: inside
// W[e][d] = sum_j v_j[e] (a^(n-1-j) k_j[d]) of a (chunk, head), float32.  A wave takes two tiles of 16 value channels at a
// time.  Operands of v_mfma_f32_16x16x32_bf16 (r = lane % 16, g = lane / 16): A lane holds A[r][8g..8g+7], B lane holds
// B[8g..8g+7][r], C lane holds C[4g..4g+3][r].
template <bool VLO>
__global__ __launch_bounds__(256) void decay_inside_kernel(const bf16_t* __restrict__ kt_ws, const bf16_t* __restrict__ vt_ws, int n_heads, int dim,
                                                           int vdim, int chunk0, float* __restrict__ w_ws) {
  const int c = blockIdx.x, h = blockIdx.y, wave = threadIdx.x / 64, lane = threadIdx.x % 64, r = lane % 16, g = lane / 16;
  const size_t slab = static_cast<size_t>(chunk0 + c) * n_heads + h;
  const bf16_t* kt = kt_ws + slab * dim * kChunk * 2;
  const bf16_t* vt = vt_ws + slab * vdim * kChunk * (VLO ? 2 : 1);
  float* w = w_ws + (static_cast<size_t>(c) * n_heads + h) * vdim * dim;
  const int n_e = vdim / 16, n_d = dim / 16;
  // (waves without a pair of value tiles of their own share the key tiles of the others')
  const int e_pairs = (n_e + 1) / 2, e_waves = min(4, e_pairs), d_waves = 4 / e_waves;
  const int ew = wave % e_waves, dw = wave / e_waves;
  if (dw >= d_waves) return;
  for (int ep = ew; ep < e_pairs; ep += e_waves) {
    Pair a[2][2];
#pragma unroll
    for (int x = 0; x < 2; ++x) {
      const int e = min(2 * ep + x, n_e - 1) * 16 + r;
#pragma unroll
      for (int u = 0; u < 2; ++u) {
        const bf16_t* p = vt + (static_cast<size_t>(e) * (kChunk / 8) + 4 * u + g) * (VLO ? 16 : 8);
        a[x][u].hi.u = *reinterpret_cast<const u32x4_t*>(p);
        if (VLO) a[x][u].lo.u = *reinterpret_cast<const u32x4_t*>(p + 8);
      }
    }
    for (int dt = dw; dt < n_d; dt += d_waves) {
      f32x4_t acc[2] = {f32x4_t{0.f, 0.f, 0.f, 0.f}, f32x4_t{0.f, 0.f, 0.f, 0.f}};
#pragma unroll
      for (int u = 0; u < 2; ++u) {
        const Pair b = load_pair(kt + (static_cast<size_t>(16 * dt + r) * (kChunk / 8) + 4 * u + g) * 16);
#pragma unroll
        for (int x = 0; x < 2; ++x) {
          acc[x] = mma(a[x][u].hi, b.lo, mma(a[x][u].hi, b.hi, acc[x]));
          if (VLO) acc[x] = mma(a[x][u].lo, b.hi, acc[x]);
        }
      }
#pragma unroll
      for (int x = 0; x < 2; ++x)
        if (2 * ep + x < n_e) {
#pragma unroll
          for (int i = 0; i < 4; ++i) w[static_cast<size_t>((2 * ep + x) * 16 + 4 * g + i) * dim + 16 * dt + r] = acc[x][i];
        }
    }
  }
}

// ---------------------------------------------------------------------------------------- chunks: across
// A thread eight neighbouring key channels of one value channel: S = a^n S + W along the request's chunks within [chunk0,
// chunk0 + n_chunks); the memory before a chunk replaces the chunk's W as [8 hi | 8 lo].
__global__ __launch_bounds__(256) void decay_across_kernel(float* __restrict__ w_ws, float* __restrict__ state, const int32_t* __restrict__ state_slots,
                                                           const int32_t* __restrict__ seq_chunk0, const int32_t* __restrict__ chunks, int chunk0,
                                                           int n_chunks, int n_heads, int dim, int vdim, const float* __restrict__ decay) {
  const int seq = blockIdx.z, h = blockIdx.y;
  const int first = max(seq_chunk0[seq], chunk0), last = min(seq_chunk0[seq + 1], chunk0 + n_chunks);
  const int i = blockIdx.x * 256 + threadIdx.x, pieces = dim / 8;
  if (first >= last || i >= vdim * pieces) return;
  const int e = i / pieces, d = 8 * (i % pieces);
  float* S_head = state + (static_cast<size_t>(state_slots[seq]) * n_heads + h) * dim * vdim;
  float S[8];
#pragma unroll
  for (int x = 0; x < 8; ++x) S[x] = S_head[static_cast<size_t>(d + x) * vdim + e];
  const size_t step = static_cast<size_t>(n_heads) * vdim * dim;
  float* w = w_ws + (static_cast<size_t>(first - chunk0) * n_heads + h) * vdim * dim + static_cast<size_t>(e) * dim + d;
  const float a = decay[h], a_whole = powf(a, static_cast<float>(kChunk));
  // four chunks' sums asked for at a time
  for (int c0 = first; c0 < last; c0 += 4) {
    float4 lo[4], hi[4];
#pragma unroll
    for (int j = 0; j < 4; ++j)
      if (c0 + j < last) {
        lo[j] = *reinterpret_cast<const float4*>(w + j * step);
        hi[j] = *reinterpret_cast<const float4*>(w + j * step + 4);
      }
#pragma unroll
    for (int j = 0; j < 4; ++j)
      if (c0 + j < last) {
        const int n = chunks[3 * (c0 + j) + 2];
        const float an = n == kChunk ? a_whole : powf(a, static_cast<float>(n));
        u32x4_t h8, l8;
        split8(S, h8, l8);
        *reinterpret_cast<float4*>(w + j * step) = make_float4(__uint_as_float(h8[0]), __uint_as_float(h8[1]), __uint_as_float(h8[2]), __uint_as_float(h8[3]));
        *reinterpret_cast<float4*>(w + j * step + 4) = make_float4(__uint_as_float(l8[0]), __uint_as_float(l8[1]), __uint_as_float(l8[2]), __uint_as_float(l8[3]));
        S[0] = fmaf(an, S[0], lo[j].x); S[1] = fmaf(an, S[1], lo[j].y); S[2] = fmaf(an, S[2], lo[j].z); S[3] = fmaf(an, S[3], lo[j].w);
        S[4] = fmaf(an, S[4], hi[j].x); S[5] = fmaf(an, S[5], hi[j].y); S[6] = fmaf(an, S[6], hi[j].z); S[7] = fmaf(an, S[7], hi[j].w);
      }
    w += 4 * step;
  }
#pragma unroll
  for (int x = 0; x < 8; ++x) S_head[static_cast<size_t>(d + x) * vdim + e] = S[x];
}

// ---------------------------------------------------------------------------------------- chunks: out
// o of a (chunk, head).  A wave owns CT tiles of 16 tokens (the columns) and, with CT = 2, every other tile of 16 value
// channels: out^T = (S^T q a^(i+1)) + v^T P^T with P^T[j][i] = a^(i-j) k_j . q_i.  The 16 rows of the two score products of a
// group of 32 keys stand for keys 8 (row / 4) + row % 4 and 4 more, so that afterwards lane group g holds keys 8g .. 8g+7 in
// order, as the second product's operand wants them.
template <int KS, int CT, bool VLO>
__global__ __launch_bounds__(256) void decay_out_kernel(const bf16_t* __restrict__ q_ws, const bf16_t* __restrict__ k_ws, const bf16_t* __restrict__ vt_ws,
                                                        const float* __restrict__ s_ws, const int32_t* __restrict__ chunks, int chunk0, int n_heads,
                                                        int vdim, const float* __restrict__ decay, float* __restrict__ out) {
  constexpr int dim = 32 * KS, pieces = dim / 8;
  __shared__ float power[kChunk + 1];
  const int c = blockIdx.x, h = blockIdx.y, wave = threadIdx.x / 64, lane = threadIdx.x % 64, r = lane % 16, g = lane / 16;
  const int tok0 = chunks[3 * (chunk0 + c) + 1], n = chunks[3 * (chunk0 + c) + 2];
  if (threadIdx.x <= kChunk) power[threadIdx.x] = powf(decay[h], static_cast<float>(threadIdx.x));
  __syncthreads();
  const int col0 = 16 * CT * (wave / CT), e_first = wave % CT;  // first token of this wave; its first tile of value channels
  if (col0 >= n) return;
  const size_t slab = static_cast<size_t>(chunk0 + c) * n_heads + h;
  const bf16_t* q = q_ws + slab * kChunk * dim * 2;
  const bf16_t* k = k_ws + slab * kChunk * dim * 2;
  const bf16_t* vt = vt_ws + slab * vdim * kChunk * (VLO ? 2 : 1);
  const bf16_t* st = reinterpret_cast<const bf16_t*>(s_ws + (static_cast<size_t>(c) * n_heads + h) * vdim * dim);
  Pair qf[CT][KS];
#pragma unroll
  for (int t = 0; t < CT; ++t)
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) qf[t][ks] = load_pair(q + (static_cast<size_t>(col0 + 16 * t + r) * pieces + 4 * ks + g) * 16);
  const int groups = (min(n, col0 + 16 * CT) + 31) / 32;  // of 32 keys, as far as this wave's tokens see
  Pair pf[CT][2];
#pragma unroll
  for (int u = 0; u < 2; ++u) {
    float p[CT][8];
#pragma unroll
    for (int sb = 0; sb < 2; ++sb) {
      f32x4_t s[CT];
#pragma unroll
      for (int t = 0; t < CT; ++t) s[t] = f32x4_t{0.f, 0.f, 0.f, 0.f};
      if (u < groups) {
        const bf16_t* krow = k + static_cast<size_t>(32 * u + 8 * (r / 4) + 4 * sb + r % 4) * pieces * 16;
#pragma unroll
        for (int ks = 0; ks < KS; ++ks) {
          const Pair a = load_pair(krow + (4 * ks + g) * 16);
#pragma unroll
          for (int t = 0; t < CT; ++t) s[t] = mma_pairs(a, qf[t][ks], s[t]);
        }
      }
#pragma unroll
      for (int t = 0; t < CT; ++t)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int back = col0 + 16 * t + r - (32 * u + 8 * g + 4 * sb + i);
          p[t][4 * sb + i] = back >= 0 ? s[t][i] * power[max(back, 0)] : 0.f;
        }
    }
#pragma unroll
    for (int t = 0; t < CT; ++t) split8(p[t], pf[t][u].hi.u, pf[t][u].lo.u);
  }
  float before[CT];  // what the memory before the chunk has decayed to at the column's token
#pragma unroll
  for (int t = 0; t < CT; ++t) before[t] = power[col0 + 16 * t + r + 1];
  // (a tile's memory and values are asked for while the tile before is worked on)
  const int n_e = vdim / 16;
  Pair sf[KS], vf[2];
  auto ask = [&](int et) {
    const bf16_t* srow = st + static_cast<size_t>(16 * et + r) * pieces * 16;
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) sf[ks] = load_pair(srow + (4 * ks + g) * 16);
#pragma unroll
    for (int u = 0; u < 2; ++u) {
      const bf16_t* p = vt + (static_cast<size_t>(16 * et + r) * (kChunk / 8) + 4 * u + g) * (VLO ? 16 : 8);
      vf[u].hi.u = *reinterpret_cast<const u32x4_t*>(p);
      if (VLO) vf[u].lo.u = *reinterpret_cast<const u32x4_t*>(p + 8);
    }
  };
  if (e_first < n_e) ask(e_first);
  for (int et = e_first; et < n_e; et += CT) {
    f32x4_t acc[CT];
#pragma unroll
    for (int t = 0; t < CT; ++t) acc[t] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    Pair s_now[KS], v_now[2];
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) s_now[ks] = sf[ks];
    v_now[0] = vf[0], v_now[1] = vf[1];
    if (et + CT < n_e) ask(et + CT);
#pragma unroll
    for (int ks = 0; ks < KS; ++ks)
#pragma unroll
      for (int t = 0; t < CT; ++t) acc[t] = mma_pairs(s_now[ks], qf[t][ks], acc[t]);
#pragma unroll
    for (int t = 0; t < CT; ++t) acc[t] *= before[t];
#pragma unroll
    for (int u = 0; u < 2; ++u)
      if (u < groups) {
#pragma unroll
        for (int t = 0; t < CT; ++t) {
          acc[t] = mma(v_now[u].hi, pf[t][u].lo, mma(v_now[u].hi, pf[t][u].hi, acc[t]));
          if (VLO) acc[t] = mma(v_now[u].lo, pf[t][u].hi, acc[t]);
        }
      }
#pragma unroll
    for (int t = 0; t < CT; ++t) {
      const int i = col0 + 16 * t + r;
      if (i < n)
        *reinterpret_cast<f32x4_t*>(out + (static_cast<size_t>(tok0 + i) * n_heads + h) * vdim + 16 * et + 4 * g) = acc[t];
    }
  }
}

// Whether the chunks' kernels take these sizes (bfloat16 rows; the rest of the spans go to the plain scan).
extern "C" int yk_decay_scan_chunks_ok(int dim, int vdim, int rot, int interleaved) {
  return (dim == 32 || dim == 64 || dim == 128 || dim == 256) && vdim % 16 == 0 && vdim <= 512 && rot % (interleaved ? 8 : 16) == 0 ? 1 : 0;
}
// bytes of scratch: the prepared operands of all chunks, and the sums of `slab_chunks` of them at a time
static size_t decay_operand_elems(int n_chunks, int n_heads, int dim, int vdim, int silu) {
  return static_cast<size_t>(n_chunks) * n_heads * kChunk * (3 * 2 * static_cast<size_t>(dim) + (silu ? 2 : 1) * static_cast<size_t>(vdim));
}
extern "C" size_t yk_decay_scan_chunks_bytes(int n_chunks, int slab_chunks, int n_heads, int dim, int vdim, int silu) {
  return decay_operand_elems(n_chunks, n_heads, dim, vdim, silu) * 2 + static_cast<size_t>(slab_chunks) * n_heads * dim * vdim * 4;
}

extern "C" int yk_decay_scan_chunks(const void* src, int src_stride, int n_heads, int dim, int vdim, float* state, const int32_t* state_slots,
                                    int n_seqs, const int32_t* chunks, int n_chunks, const int32_t* seq_chunk0, int slab_chunks,
                                    const int32_t* positions, const float* cos_t, const float* sin_t, int rot, int interleaved, int max_pos,
                                    float k_scale, int silu, const float* decay, void* workspace, size_t workspace_bytes, float* out,
                                    hipStream_t stream) {
  YK_REQUIRE(n_seqs >= 0 && n_chunks >= 0 && n_heads > 0 && src_stride >= n_heads * (2 * dim + vdim), "decay_scan_chunks: bad sizes");
  YK_REQUIRE(yk_decay_scan_chunks_ok(dim, vdim, rot, interleaved), "decay_scan_chunks: sizes the chunks' kernels do not take");
  YK_REQUIRE(rot <= dim && (rot == 0 || (cos_t != nullptr && sin_t != nullptr && max_pos > 0)) && positions != nullptr, "decay_scan_chunks: rotary tables missing");
  auto al16 = [](const void* p) { return reinterpret_cast<uintptr_t>(p) % 16 == 0; };
  YK_REQUIRE(src_stride % 8 == 0 && al16(src) && al16(workspace) && al16(out), "decay_scan_chunks: rows must be 16-byte aligned");
  YK_REQUIRE(n_heads <= 65535 && n_seqs <= 65535 && slab_chunks >= 1, "decay_scan_chunks: too many heads or requests for one launch");
  YK_REQUIRE(workspace_bytes >= yk_decay_scan_chunks_bytes(n_chunks, slab_chunks, n_heads, dim, vdim, silu), "decay_scan_chunks: workspace too small");
  if (n_chunks == 0 || n_seqs == 0) return 0;
  const Inputs in{positions, cos_t, sin_t, rot, interleaved, max_pos, k_scale, silu};
  const size_t rows = static_cast<size_t>(n_chunks) * n_heads * kChunk * dim * 2;
  bf16_t* q_ws = static_cast<bf16_t*>(workspace);
  bf16_t* k_ws = q_ws + rows;
  bf16_t* kt_ws = k_ws + rows;
  bf16_t* vt_ws = kt_ws + rows;
  float* w_ws = reinterpret_cast<float*>(q_ws + decay_operand_elems(n_chunks, n_heads, dim, vdim, silu));
  {
    const dim3 grid(n_chunks, n_heads, 2 * ((dim + kPrepare - 1) / kPrepare) + (vdim + kPrepare - 1) / kPrepare);
    auto kern = silu ? decay_prepare_kernel<true> : decay_prepare_kernel<false>;
    kern<<<grid, 256, 0, stream>>>(static_cast<const bf16_t*>(src), src_stride, n_heads, dim, vdim, decay, chunks, in, q_ws, k_ws, kt_ws, vt_ws);
    if (yk_check_launch("decay_prepare")) return -1;
  }
  for (int c0 = 0; c0 < n_chunks; c0 += slab_chunks) {
    const int nc = std::min(slab_chunks, n_chunks - c0);
    const dim3 grid(nc, n_heads);
    if (silu) decay_inside_kernel<true><<<grid, 256, 0, stream>>>(kt_ws, vt_ws, n_heads, dim, vdim, c0, w_ws);
    else decay_inside_kernel<false><<<grid, 256, 0, stream>>>(kt_ws, vt_ws, n_heads, dim, vdim, c0, w_ws);
    if (yk_check_launch("decay_inside")) return -1;
    decay_across_kernel<<<dim3((vdim * (dim / 8) + 255) / 256, n_heads, n_seqs), 256, 0, stream>>>(w_ws, state, state_slots, seq_chunk0, chunks, c0, nc,
                                                                                                  n_heads, dim, vdim, decay);
    if (yk_check_launch("decay_across")) return -1;
#define YK_OUT(KS, CT)                                                                                                                \
  if (dim == 32 * KS) {                                                                                                               \
    if (silu) decay_out_kernel<KS, CT, true><<<grid, 256, 0, stream>>>(q_ws, k_ws, vt_ws, w_ws, chunks, c0, n_heads, vdim, decay, out); \
    else decay_out_kernel<KS, CT, false><<<grid, 256, 0, stream>>>(q_ws, k_ws, vt_ws, w_ws, chunks, c0, n_heads, vdim, decay, out);    \
  }
    YK_OUT(1, 2)
    YK_OUT(2, 2)
    YK_OUT(4, 2)
    YK_OUT(8, 1)
#undef YK_OUT
    if (yk_check_launch("decay_out")) return -1;
  }
  return 0;
}

// ---------------------------------------------------------------------------------------- single tokens
// LANES lanes side by side over the columns (four each), 256 / LANES groups over the rows.
constexpr int kStepRows = 8;  // rows of a thread asked for at a time
template <typename T, int LANES>
__global__ __launch_bounds__(256) void decay_step_kernel(const T* __restrict__ src, int src_stride, int n_heads, int dim, int vdim,
                                                         float* __restrict__ state, const int32_t* __restrict__ seq_qstart,
                                                         const int32_t* __restrict__ state_slots, Inputs in, const float* __restrict__ decay,
                                                         float* __restrict__ out) {
  constexpr int GROUPS = 256 / LANES;
  extern __shared__ float qk[];  // q [dim], k [dim]
  __shared__ float4 part[256];
  const int seq = blockIdx.x, h = blockIdx.y, lane = threadIdx.x % LANES, group = threadIdx.x / LANES;
  const int col = (blockIdx.z * LANES + lane) * 4;
  const int n = seq_qstart[seq];
  float* S = state + (static_cast<size_t>(state_slots[seq]) * n_heads + h) * dim * vdim + col;
  float4 rows[kStepRows];
#pragma unroll
  for (int j = 0; j < kStepRows; ++j) {
    const int d = group + j * GROUPS;
    if (d < dim) rows[j] = *reinterpret_cast<const float4*>(S + static_cast<size_t>(d) * vdim);
  }
  const T* row = src + static_cast<size_t>(n) * src_stride;
  const int pos = in.rot > 0 ? min(in.positions[n], in.max_pos - 1) : 0;
  for (int i = threadIdx.x; i < 2 * dim; i += 256) {
    const int d = i % dim, is_k = i / dim;
    const T* x = row + is_k * n_heads * dim + h * dim;
    auto at = [&](int e) { const float v = to_f32<T>(x[e]); return in.silu ? act_silu(v) : v; };
    float v = at(d);
    if (d < in.rot) {
      const int half = in.rot / 2, m = in.interleaved ? d / 2 : (d < half ? d : d - half);
      const bool first = in.interleaved ? d % 2 == 0 : d < half;
      const float other = at(in.interleaved ? (first ? d + 1 : d - 1) : (first ? d + half : d - half));
      const float c = in.cos_t[static_cast<size_t>(pos) * half + m], s = in.sin_t[static_cast<size_t>(pos) * half + m];
      v = first ? rot_first(v, other, c, s) : rot_second(other, v, c, s);
    }
    qk[i] = is_k ? v * in.k_scale : v;
  }
  float v[4];
#pragma unroll
  for (int e = 0; e < 4; ++e) {
    const float x = to_f32<T>(row[2 * n_heads * dim + h * vdim + col + e]);
    v[e] = in.silu ? act_silu(x) : x;
  }
  const float a = decay[h];
  __syncthreads();
  float4 o = make_float4(0.f, 0.f, 0.f, 0.f);
  for (int d0 = 0; d0 < dim; d0 += kStepRows * GROUPS) {
    if (d0 > 0) {
#pragma unroll
      for (int j = 0; j < kStepRows; ++j) {
        const int d = d0 + group + j * GROUPS;
        if (d < dim) rows[j] = *reinterpret_cast<const float4*>(S + static_cast<size_t>(d) * vdim);
      }
    }
#pragma unroll
    for (int j = 0; j < kStepRows; ++j) {
      const int d = d0 + group + j * GROUPS;
      if (d < dim) {
        const float q = qk[d], k = qk[dim + d];
        float4 s = rows[j];
        s.x = fmaf(k, v[0], a * s.x); s.y = fmaf(k, v[1], a * s.y); s.z = fmaf(k, v[2], a * s.z); s.w = fmaf(k, v[3], a * s.w);
        *reinterpret_cast<float4*>(S + static_cast<size_t>(d) * vdim) = s;
        o.x = fmaf(q, s.x, o.x); o.y = fmaf(q, s.y, o.y); o.z = fmaf(q, s.z, o.z); o.w = fmaf(q, s.w, o.w);
      }
    }
  }
  part[threadIdx.x] = o;
  __syncthreads();
  // LANES * 4 columns, a thread each: the groups' parts in order
  if (threadIdx.x < LANES * 4) {
    const float* p = reinterpret_cast<const float*>(part) + threadIdx.x;
    float sum = 0.f;
#pragma unroll 8
    for (int y = 0; y < GROUPS; ++y) sum += p[y * LANES * 4];
    out[(static_cast<size_t>(n) * n_heads + h) * vdim + blockIdx.z * LANES * 4 + threadIdx.x] = sum;
  }
}

extern "C" int yk_decay_scan_step(const void* src, int src_stride, int dtype, int n_heads, int dim, int vdim, float* state,
                                  const int32_t* seq_qstart, const int32_t* state_slots, int n_seqs, const int32_t* positions, const float* cos_t,
                                  const float* sin_t, int rot, int interleaved, int max_pos, float k_scale, int silu, const float* decay,
                                  float* out, hipStream_t stream) {
  YK_REQUIRE(n_seqs >= 0 && n_heads > 0 && n_heads <= 65535 && dim > 0 && dim <= 4096 && vdim > 0 && src_stride >= n_heads * (2 * dim + vdim),
             "decay_scan_step: bad sizes");
  YK_REQUIRE(vdim % 4 == 0 && reinterpret_cast<uintptr_t>(state) % 16 == 0, "decay_scan_step: columns come four at a time");
  YK_REQUIRE(rot >= 0 && rot % 2 == 0 && rot <= dim && (rot == 0 || (cos_t != nullptr && sin_t != nullptr && positions != nullptr && max_pos > 0)),
             "decay_scan_step: rotary tables missing, or more elements than a head has");
  if (n_seqs == 0) return 0;
  const Inputs in{positions, cos_t, sin_t, rot, interleaved, max_pos, k_scale, silu};
  const size_t lds = 2 * static_cast<size_t>(dim) * sizeof(float);
#define YK_STEP(D, T, L)                                                                                                              \
  if (dtype == D && vdim % (4 * L) == 0) {                                                                                            \
    decay_step_kernel<T, L><<<dim3(n_seqs, n_heads, vdim / (4 * L)), 256, lds, stream>>>(static_cast<const T*>(src), src_stride, n_heads, dim, vdim, \
                                                                                         state, seq_qstart, state_slots, in, decay, out); \
    return yk_check_launch("decay_step");                                                                                             \
  }
#define YK_STEPS(D, T) YK_STEP(D, T, 16) YK_STEP(D, T, 8) YK_STEP(D, T, 4) YK_STEP(D, T, 2) YK_STEP(D, T, 1)
  YK_STEPS(YK_F32, float)
  YK_STEPS(YK_BF16, bf16_t)
#undef YK_STEPS
#undef YK_STEP
  return yk_fail("decay_scan_step: unsupported dtype");
}
