// Linear attention with a decay: S <- D S + k v^T, o = S^T q with S [dk, dv] per head, no softmax and no denominator. D is
// one fixed number per head, or (channel decay) one number per head, key channel and token that acts on the rows of S:
// alpha = sigmoid(z)^(1 / tau) with z = W_up m + bias for a narrow row m that is columns of the projection's rows too. z is
// computed where it is used (in fp32), which is cheaper than a launch that writes its rows. fp32 or bf16 projections, everything from there on and the state in fp32. q, k and v are columns of one
// projection's rows; on their way in they pass, as asked, silu (all three), a rotation of the pairs (i, i + rot / 2) among
// the first rot entries of every q and k head by the row's position, and a constant on k. A request's rows of a step are
// consecutive and in order (row_req ascends), their positions too.
//
//   linear_scan     token by token, for steps of few rows per request and for sizes that the chunked form does not take:
//                   a workgroup of four waves owns 16 value columns of one head of one request, 16 lanes per column with
//                   a sixteenth of the state rows each; the state stays in registers while the rows are walked.
//   The chunked form, for portions of prompts: with the decay fixed, C tokens move the state by
//   S' = d^C S + sum_t d^(C - 1 - t) k_t v_t^T, one product of a [dk, C] and a [C, dv] matrix, and what a token reads splits
//   into what the chunk found and what it wrote itself. A request's rows are cut into chunks of 64:
//   linear_local    per chunk, head and 128 value columns: the chunk's own sum, into a scratch array
//   linear_combine  per request, head and entry: walks the chunks in order, leaves the state in front of every chunk in
//                   the place of the chunk's sum; the last one is the request's new state
//   linear_outputs  per chunk and head: o_t = d^(t + 1) S^T q_t + sum_(s <= t) d^(t - s) (q_t . k_s) v_s, three products
//   The products of the chunked form are fp32 matrix-core instructions (v_mfma_f32_16x16x4_f32: fp32 operands, fp32
//   sums), so the two forms differ by the order of their sums only. The powers of a head's decay come from a table
//   [heads, 65] that the host computes in double.
//
// With a channel decay the chunked form is the same three steps; what takes the powers' place are products of the chunk's
// alphas, which are only ever multiplied and never divided by (a ratio of two running products overflows where a token
// forgets everything). The 64 rows are four tiles of 16; within a tile, with p_i the product of the alphas of the tile's
// rows up to i, u_j of the rows behind j, and T of all of them:
//   linear_channel_local    k_j u_j T_(later tiles) takes the place of d^(C - 1 - j) k_j; the chunk's own product per
//                           channel goes to a scratch array for linear_combine
//   linear_channel_outputs  between two tiles P[i][j] = sum_c q_ic p_ic T_c(tiles between) u_jc k_jc is one product.
//                           Within a tile, pairs are taken apart by the highest bit in which their places i > j differ:
//                           for bit s they lie in the two halves of a block of 2 s rows, and the alphas between them are the
//                           product up to i of the block's second half times the product behind j of its first half. So
//                           four products of [second halves] x [first halves], of each of which its own pairs are kept,
//                           and the diagonal q_i . k_i. A lane holds a row's entries and its 16 neighbours the other
//                           rows', so the half-block products come from each other by lane permutations.
//
// State of one request: [heads, dv, dk] (a head's matrix column by column).
#include <math.h>

#include "common.h"
#include "mfma.h"
#include "recurrence.h"

#define LIN_COLS 16
#define LIN_PARTS 16
#define LIN_ROWS 64            // rows of a chunk
#define LIN_POWERS (LIN_ROWS + 1)
#define LIN_MIDDLE 32          // a channel decay's narrow row comes in steps of this many

__device__ __forceinline__ floatx4 mfma_f32(float a, float b, floatx4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0);
}

struct LinArgs {
  const void* y;      // [rows, ld]: q (heads x dk) from q_off, k (heads x dk) from k_off, v (heads x dv) from v_off
  int ld, q_off, k_off, v_off;
  const int* positions;
  const float* cos_t;  // [positions, rot / 2]
  const float* sin_t;
  int rot, silu;
  float k_scale;
  const float* powers;  // [heads, 65]: d^0 .. d^64
  float* state;         // [slots, heads, dv, dk]
  float* out;           // [rows, ldo]: heads x dv
  int ldo;
  const int* row_req;
  const int* state_slots;
  int n_rows, heads, dk, dv;
  // the chunked form
  const int* requests;  // [requests, 3]: first row, rows, first chunk
  const int* chunks;    // [chunks, 2]: first row, rows
  float* before;        // [chunks, heads, dv, dk]: a chunk's own sum, then the state in front of it
  // channel decay (powers are then unused)
  int m_off, middle;    // the narrow row: columns m_off .. + middle of y (a multiple of LIN_MIDDLE, filled up with zeros)
  int rank;             // what of it is not filling
  const void* w_up;     // [heads x dk, middle], of y's type
  const float* b_up;    // [heads x dk]
  float inv_tau;
  float* chunk_decay;   // [chunks, heads, dk]: the product of a chunk's alphas
};

// sigmoid(z)^(1 / tau), through its logarithm (log sigmoid(z) = min(z, 0) - log(1 + exp(-|z|)), which no z overflows)
template <typename T>
__device__ __forceinline__ float channel_alpha(float z, float inv_tau);
template <>
__device__ __forceinline__ float channel_alpha<float>(float z, float inv_tau) {
  return expf((fminf(z, 0.f) - log1pf(expf(-fabsf(z)))) * inv_tau);
}
template <>
__device__ __forceinline__ float channel_alpha<bf16_t>(float z, float inv_tau) {
  // the hardware's exp2 and log2. A decay near 1 acts on hundreds of tokens, so what 1 + x loses of a small x = exp(-|z|) is
  // made good: log(1 + x) = x log(u) / (u - 1) with u = 1 + x as rounded, and x itself where u is 1
  const float z2 = 1.4426950408889634f * z;
  const float x = __builtin_amdgcn_exp2f(-fabsf(z2)), u = 1.0f + x, d = u - 1.0f;
  const float l = d == 0.f ? 1.4426950408889634f * x : __builtin_amdgcn_logf(u) * x * __builtin_amdgcn_rcpf(d);
  return __builtin_amdgcn_exp2f((fminf(z2, 0.f) - l) * inv_tau);
}

// bf16 inputs: the hardware's exp2 and reciprocal (each within a unit or two of the last place in fp32)
template <typename T>
__device__ __forceinline__ float lin_act(float z, int silu);
template <>
__device__ __forceinline__ float lin_act<float>(float z, int silu) { return silu ? z / (1.0f + expf(-z)) : z; }
template <>
__device__ __forceinline__ float lin_act<bf16_t>(float z, int silu) {
  return silu ? z * __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-1.4426950408889634f * z)) : z;
}

template <typename T>
struct Raw4;  // four neighbouring elements as they lie in memory
template <>
struct Raw4<float> {
  float4 v;
  __device__ __forceinline__ void load(const float* p) { v = *(const float4*)p; }
  __device__ __forceinline__ float get(int e) const { return e == 0 ? v.x : e == 1 ? v.y : e == 2 ? v.z : v.w; }
};
template <>
struct Raw4<bf16_t> {
  uint2 v;
  __device__ __forceinline__ void load(const bf16_t* p) { v = *(const uint2*)p; }
  __device__ __forceinline__ float get(int e) const {
    const uint32_t w = e < 2 ? v.x : v.y;
    return __uint_as_float((e & 1) ? (w & 0xffff0000u) : (w << 16));
  }
};

// thread = cw * 16 + part: column blockIdx.z * 16 + cw, state rows part * E .. + E. C: rows staged at a time
template <typename T, int E, int C, bool ROT, bool CHAN>
__global__ __launch_bounds__(256) void linear_scan_kernel(LinArgs A) {
  constexpr int NP = LIN_PARTS * E;          // the key size, padded with zeros
  constexpr int VAT = (CHAN ? 3 : 2) * NP;
  constexpr int ROWF = VAT + LIN_COLS + 4;  // q | k (| alpha) | v of the workgroup's columns | -
  constexpr int NQK = (C * 2 * NP + 255) / 256;
  constexpr int NAL = (C * NP + 255) / 256;
  __shared__ __align__(16) float sm[C * ROWF];
  const int tid = threadIdx.x;
  const int part = tid & 15, cw = tid >> 4;
  const int req = blockIdx.x, h = blockIdx.y;
  const int col0 = blockIdx.z * LIN_COLS;
  const int col = col0 + cw;
  const bool col_on = col < A.dv;
  int lo, n;
  rows_of_request(A.row_req, A.n_rows, req, lo, n);
  if (n == 0) return;
  const int dk = A.dk;
  const int i0 = part * E;
  float* S_at = A.state + ((size_t)A.state_slots[req] * A.heads + h) * dk * A.dv;
  float S[E];
  // every lane loads from a place that exists and drops what it does not own, so that the loads are in flight together
  const bool wide = E >= 4 && (dk & 3) == 0;  // then a lane's entries start on 16 bytes and end with the column
  if (wide) {
#pragma unroll
    for (int e = 0; e < E; e += 4) {
      const bool own = col_on && i0 + e < dk;
      const float4 s = *reinterpret_cast<const float4*>(S_at + (own ? (size_t)col * dk + i0 + e : 0));
      S[e] = own ? s.x : 0.f;
      S[(e + 1) % E] = own ? s.y : 0.f;
      S[(e + 2) % E] = own ? s.z : 0.f;
      S[(e + 3) % E] = own ? s.w : 0.f;
    }
  } else {
#pragma unroll
    for (int e = 0; e < E; ++e) {
      const bool own = col_on && i0 + e < dk;
      const float s = S_at[own ? (size_t)col * dk + i0 + e : 0];
      S[e] = own ? s : 0.f;
    }
  }
  const T* y = (const T*)A.y;
  const int half = A.rot >> 1;
  const int pos0 = ROT ? A.positions[lo] : 0;
  // four entries of the narrow row per load where it lies on them
  const bool mid_wide = CHAN && ((A.ld | A.m_off) & 3) == 0 && ((uintptr_t)A.y % (4 * sizeof(T))) == 0 && ((uintptr_t)A.w_up % (4 * sizeof(T))) == 0;
  const float d = CHAN ? 0.f : A.powers[(size_t)h * LIN_POWERS + 1];
  const size_t q_at = (size_t)A.q_off + (size_t)h * dk, k_at = (size_t)A.k_off + (size_t)h * dk;
  const size_t v_at = (size_t)A.v_off + (size_t)h * A.dv + col0;
  for (int r0 = 0; r0 < n; r0 += C) {
    const int have = min(C, n - r0);
    if (r0) __syncthreads();  // the rows before have been read
#pragma unroll
    for (int j = 0; j < NQK; ++j) {
      const int idx = tid + 256 * j;
      if (C * 2 * NP % 256 && idx >= C * 2 * NP) break;
      const int t = idx / (2 * NP), w = idx % (2 * NP);
      const int i = w % NP;
      const bool own = t < have && i < dk;
      const T* row = y + (size_t)(lo + r0 + (own ? t : 0)) * A.ld + (w < NP ? q_at : k_at);
      float p = lin_act<T>(ldf(row, own ? i : 0), A.silu);
      if (ROT) {
        const bool turns = own && i < A.rot;
        const int f = turns ? (i < half ? i : i - half) : 0;
        const float o = lin_act<T>(ldf(row, turns ? (i < half ? i + half : i - half) : 0), A.silu);
        const size_t at = (size_t)(pos0 + r0 + (own ? t : 0)) * half + f;
        const float c = A.cos_t[at], s = A.sin_t[at];
        if (turns) p = i < half ? p * c - o * s : p * c + o * s;
      }
      if (w >= NP) p *= A.k_scale;
      sm[t * ROWF + w] = own ? p : 0.f;
    }
    if (CHAN) {
#pragma unroll
      for (int j = 0; j < NAL; ++j) {
        const int idx = tid + 256 * j;
        if (C * NP % 256 && idx >= C * NP) break;
        const int t = idx / NP, i = idx % NP;
        const bool own = t < have && i < dk;
        const T* m = y + (size_t)(lo + r0 + (own ? t : 0)) * A.ld + A.m_off;
        const T* w = (const T*)A.w_up + ((size_t)h * dk + (own ? i : 0)) * A.middle;
        float z = A.b_up[(size_t)h * dk + (own ? i : 0)];
        if (mid_wide) {
          for (int k0 = 0; k0 < A.rank; k0 += 16) {
            Raw4<T> mu[4], wu[4];
#pragma unroll
            for (int k = 0; k < 4; ++k) mu[k].load(m + k0 + 4 * k), wu[k].load(w + k0 + 4 * k);
#pragma unroll
            for (int k = 0; k < 4; ++k)
#pragma unroll
              for (int e = 0; e < 4; ++e) z = fmaf(mu[k].get(e), wu[k].get(e), z);
          }
        } else {
          for (int k = 0; k < A.rank; ++k) z = fmaf(ldf(m, k), ldf(w, k), z);
        }
        sm[t * ROWF + 2 * NP + i] = own ? channel_alpha<T>(z, A.inv_tau) : 0.f;
      }
    }
    if (tid < C * LIN_COLS) {
      const int t = tid / LIN_COLS, cc = tid % LIN_COLS;
      const bool own = t < have && col0 + cc < A.dv;
      const float p = lin_act<T>(ldf(y + (size_t)(lo + r0 + (own ? t : 0)) * A.ld + v_at, own ? cc : 0), A.silu);
      sm[t * ROWF + VAT + cc] = own ? p : 0.f;
    }
    __syncthreads();
    for (int t = 0; t < have; ++t) {
      const float* row = sm + t * ROWF;
      const float v = row[VAT + cw];
      float o = 0.f;
#pragma unroll
      for (int e = 0; e < E; ++e) {
        S[e] = fmaf(v, row[NP + i0 + e], (CHAN ? row[2 * NP + i0 + e] : d) * S[e]);
        o = fmaf(S[e], row[i0 + e], o);
      }
      o = row16_sum(o);
      if (part == 0 && col_on) A.out[(size_t)(lo + r0 + t) * A.ldo + (size_t)h * A.dv + col] = o;
    }
  }
  if (wide) {
#pragma unroll
    for (int e = 0; e < E; e += 4)
      if (col_on && i0 + e < dk)
        *reinterpret_cast<float4*>(S_at + (size_t)col * dk + i0 + e) = make_float4(S[e], S[(e + 1) % E], S[(e + 2) % E], S[(e + 3) % E]);
  } else {
#pragma unroll
    for (int e = 0; e < E; ++e)
      if (col_on && i0 + e < dk) S_at[(size_t)col * dk + i0 + e] = S[e];
  }
}

// ---------------------------------------------------------------------------------------------------------------------
// the chunked form: dk and dv in multiples of 16 up to 256, rot in multiples of 8, rows and offsets on 4 elements

// Two groups of four entries of a q or k head that the same thread brings in: entries i1 .. + 4 and i2 .. + 4. Below rot / 2
// they are the two sides of four turned pairs, beyond it neighbours that pass unturned.
template <typename T, bool ROT>
struct HeadUnit {
  Raw4<T> a, b;
  float4 c, s;
  int i1, i2;
  bool turns;
  __device__ __forceinline__ void load(const T* head, int u, int rot, const float* cos_row, const float* sin_row) {
    const int half = rot >> 1;
    turns = ROT && u * 4 < half;
    i1 = turns ? u * 4 : rot + 2 * (u * 4 - half);
    i2 = turns ? i1 + half : i1 + 4;
    a.load(head + i1);
    b.load(head + i2);
    if (ROT) {
      const int f = turns ? u * 4 : 0;
      c = *(const float4*)(cos_row + f);
      s = *(const float4*)(sin_row + f);
    }
  }
  __device__ __forceinline__ void store(float* row, bool on, int silu, float mul) const {
    float p[4], q[4];
    const float cc[4] = {c.x, c.y, c.z, c.w}, ss[4] = {s.x, s.y, s.z, s.w};
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      p[e] = lin_act<T>(a.get(e), silu);
      q[e] = lin_act<T>(b.get(e), silu);
      if (ROT && turns) {
        const float u = p[e], v = q[e];
        p[e] = u * cc[e] - v * ss[e];
        q[e] = v * cc[e] + u * ss[e];
      }
      p[e] = on ? p[e] * mul : 0.f;
      q[e] = on ? q[e] * mul : 0.f;
    }
    *(float4*)(row + i1) = float4{p[0], p[1], p[2], p[3]};
    *(float4*)(row + i2) = float4{q[0], q[1], q[2], q[3]};
  }
};

// grid (chunk, head, 128 value columns), eight waves. Wave w sums the state rows of its DT tiles of 16 (w % 4) for four
// tiles of value columns (w / 4); lane l of a tile holds rows 4 (l / 16) .. + 4 of column l % 16.
#define LIN_LOCAL_COLS 128
template <typename T, int DT, bool ROT>
__global__ __launch_bounds__(512) void linear_local_kernel(LinArgs A) {
  constexpr int DKP = DT * 64;
  constexpr int KLD = DKP + 16;  // neighbouring rows of 16 entries lie in different banks
  constexpr int VLD = LIN_LOCAL_COLS + 16;
  constexpr int UN = DKP / 8;
  constexpr int NU = UN * LIN_ROWS / 512;
  __shared__ __align__(16) float Ks[LIN_ROWS * KLD];
  __shared__ __align__(16) float Vs[LIN_ROWS * VLD];
  const int tid = threadIdx.x;
  const int wave = tid >> 6, lane = tid & 63, l16 = lane & 15, g = lane >> 4;
  const int c = blockIdx.x, h = blockIdx.y, col0 = blockIdx.z * LIN_LOCAL_COLS;
  const int lo = A.chunks[c * 2], have = A.chunks[c * 2 + 1];
  const int dk = A.dk, dv = A.dv, units = dk >> 3;
  const int vcols = min(LIN_LOCAL_COLS, dv - col0);
  const float* pw = A.powers + (size_t)h * LIN_POWERS;
  const T* y = (const T*)A.y;
  const T* kh = y + A.k_off + (size_t)h * dk;
  const T* vh = y + A.v_off + (size_t)h * dv + col0;
  const int pos0 = ROT ? A.positions[lo] : 0;
  const int half = A.rot >> 1;
  HeadUnit<T, ROT> ku[NU];
  Raw4<T> vu[4];
  float vw[4];
  // rows and columns beyond the chunk's are read from its last ones and dropped
#pragma unroll
  for (int j = 0; j < NU; ++j) {
    const int idx = tid + 512 * j;
    const int t = min(idx / UN, have - 1), u = min(idx % UN, units - 1);
    ku[j].load(kh + (size_t)(lo + t) * A.ld, u, A.rot, ROT ? A.cos_t + (size_t)(pos0 + t) * half : nullptr,
               ROT ? A.sin_t + (size_t)(pos0 + t) * half : nullptr);
  }
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    const int t = (tid >> 5) + 16 * j;
    vu[j].load(vh + (size_t)(lo + min(t, have - 1)) * A.ld + min((tid & 31) * 4, vcols - 4));
    vw[j] = pw[max(have - 1 - t, 0)];
  }
#pragma unroll
  for (int j = 0; j < NU; ++j) {
    const int idx = tid + 512 * j;
    const int t = idx / UN, u = idx % UN;
    float* row = Ks + t * KLD;
    if (u < units) {
      ku[j].store(row, t < have, A.silu, A.k_scale);
    } else {  // the padding behind the key size
      *(float4*)(row + u * 8) = float4{0.f, 0.f, 0.f, 0.f};
      *(float4*)(row + u * 8 + 4) = float4{0.f, 0.f, 0.f, 0.f};
    }
  }
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    const int t = (tid >> 5) + 16 * j;
    const bool on = t < have && (tid & 31) * 4 < vcols;
    float v[4];
#pragma unroll
    for (int e = 0; e < 4; ++e) v[e] = on ? lin_act<T>(vu[j].get(e), A.silu) * vw[j] : 0.f;
    *(float4*)(Vs + t * VLD + (tid & 31) * 4) = float4{v[0], v[1], v[2], v[3]};
  }
  __syncthreads();
  const int dk_tile = (wave & 3) * DT, v_tile = (wave >> 2) * 4;
  if (dk_tile * 16 >= dk || v_tile * 16 >= vcols) return;  // nothing of this wave's is in the matrix
  floatx4 S[DT][4];
#pragma unroll
  for (int j = 0; j < DT; ++j)
#pragma unroll
    for (int n = 0; n < 4; ++n) S[j][n] = floatx4{0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
  for (int t0 = 0; t0 < have; t0 += 4) {
    float a[DT], b[4];
#pragma unroll
    for (int j = 0; j < DT; ++j) a[j] = Ks[(t0 + g) * KLD + (dk_tile + j) * 16 + l16];
#pragma unroll
    for (int n = 0; n < 4; ++n) b[n] = Vs[(t0 + g) * VLD + (v_tile + n) * 16 + l16];
#pragma unroll
    for (int n = 0; n < 4; ++n)
      if ((v_tile + n) * 16 < vcols) {
#pragma unroll
        for (int j = 0; j < DT; ++j) S[j][n] = mfma_f32(a[j], b[n], S[j][n]);
      }
  }
#pragma unroll
  for (int j = 0; j < DT; ++j) {
    const int i = (dk_tile + j) * 16 + 4 * g;
    if (i >= dk) continue;
#pragma unroll
    for (int n = 0; n < 4; ++n)
      if ((v_tile + n) * 16 < vcols)
        *(floatx4*)(A.before + (((size_t)c * A.heads + h) * dv + col0 + (v_tile + n) * 16 + l16) * dk + i) = S[j][n];
  }
}

// grid (1,024 entries, head, request): a thread carries four entries of the state through the request's chunks
template <bool CHAN>
__global__ __launch_bounds__(256) void linear_combine_kernel(LinArgs A) {
  constexpr int AHEAD = 8;
  const int h = blockIdx.y, req = blockIdx.z;
  const size_t n = (size_t)A.dk * A.dv;
  const size_t i = ((size_t)blockIdx.x * 256 + threadIdx.x) * 4;
  if (i >= n) return;
  const int rows = A.requests[req * 3 + 1], c0 = A.requests[req * 3 + 2];
  if (rows <= 0) return;
  const int chunks = (rows + LIN_ROWS - 1) / LIN_ROWS;
  const float* pw = A.powers + (size_t)h * LIN_POWERS;
  const float d_full = CHAN ? 0.f : pw[LIN_ROWS], d_last = CHAN ? 0.f : pw[rows - (chunks - 1) * LIN_ROWS];
  const float* cd = CHAN ? A.chunk_decay + ((size_t)c0 * A.heads + h) * A.dk + i % A.dk : nullptr;  // dk is a multiple of 16
  const size_t cd_step = (size_t)A.heads * A.dk;
  float* st = A.state + ((size_t)A.state_slots[req] * A.heads + h) * n + i;
  const size_t step = (size_t)A.heads * n;
  float* buf = A.before + ((size_t)c0 * A.heads + h) * n + i;
  floatx4 S = *(const floatx4*)st;
  for (int c = 0; c < chunks; c += AHEAD) {
    floatx4 kv[AHEAD], dc[AHEAD];
#pragma unroll
    for (int j = 0; j < AHEAD; ++j) {
      kv[j] = *(const floatx4*)(buf + (size_t)min(c + j, chunks - 1) * step);
      if (CHAN) dc[j] = *(const floatx4*)(cd + (size_t)min(c + j, chunks - 1) * cd_step);
    }
#pragma unroll
    for (int j = 0; j < AHEAD; ++j) {
      if (c + j >= chunks) break;
      *(floatx4*)(buf + (size_t)(c + j) * step) = S;
      if (CHAN)
        S = dc[j] * S + kv[j];
      else
        S = (c + j + 1 < chunks ? d_full : d_last) * S + kv[j];
    }
  }
  *(floatx4*)st = S;
}

// grid (chunk, head), eight waves. LDS: Q [64][dk], the ten tiles of P on and below the diagonal, K [64][dk] (later V
// [64][dv] in its place).
#define LIN_PLD 20                     // floats between the rows of a tile of P
#define LIN_PTILE (16 * LIN_PLD)
template <typename T, int DT, bool ROT>
__global__ __launch_bounds__(512) void linear_outputs_kernel(LinArgs A) {
  constexpr int DKP = DT * 64;
  constexpr int QLD = DKP + 4;
  constexpr int UN = DKP / 8;
  constexpr int NU = UN * LIN_ROWS / 512;
  constexpr int NV = 8;  // pieces of V per thread, for values of up to 256
  constexpr int KS = DKP / 16;
  extern __shared__ __align__(16) float lin_smem[];
  float* Qs = lin_smem;
  float* Ps = Qs + LIN_ROWS * QLD;
  float* Ks = Ps + 10 * LIN_PTILE;
  const int tid = threadIdx.x;
  const int wave = tid >> 6, lane = tid & 63, l16 = lane & 15, g = lane >> 4;
  const int c = blockIdx.x, h = blockIdx.y;
  const int lo = A.chunks[c * 2], have = A.chunks[c * 2 + 1];
  const int dk = A.dk, dv = A.dv, units = dk >> 3, vld = dv + 4, v4 = dv >> 2;
  const float* pw = A.powers + (size_t)h * LIN_POWERS;
  const T* y = (const T*)A.y;
  const int pos0 = ROT ? A.positions[lo] : 0;
  const int half = A.rot >> 1;
  {
    const T* head[2] = {y + A.q_off + (size_t)h * dk, y + A.k_off + (size_t)h * dk};
    HeadUnit<T, ROT> hu[2][NU];
#pragma unroll
    for (int which = 0; which < 2; ++which)
#pragma unroll
      for (int j = 0; j < NU; ++j) {
        const int idx = tid + 512 * j;
        const int t = min(idx / UN, have - 1), u = min(idx % UN, units - 1);
        hu[which][j].load(head[which] + (size_t)(lo + t) * A.ld, u, A.rot, ROT ? A.cos_t + (size_t)(pos0 + t) * half : nullptr,
                          ROT ? A.sin_t + (size_t)(pos0 + t) * half : nullptr);
      }
#pragma unroll
    for (int which = 0; which < 2; ++which)
#pragma unroll
      for (int j = 0; j < NU; ++j) {
        const int idx = tid + 512 * j;
        const int t = idx / UN, u = idx % UN;
        if (u < units) hu[which][j].store((which ? Ks : Qs) + t * QLD, t < have, A.silu, which ? A.k_scale : 1.0f);
      }
  }
  Raw4<T> vr[NV];  // in flight while P is computed
#pragma unroll
  for (int j = 0; j < NV; ++j)
    if (512 * j < LIN_ROWS * v4) {
      const int idx = tid + 512 * j;
      vr[j].load(y + (size_t)(lo + min(idx / v4, have - 1)) * A.ld + A.v_off + (size_t)h * dv + idx % v4 * 4);
    }
  // the state's part for this wave's first tile of value columns, in flight too; entries beyond dk are read from the last
  floatx4 sb[KS];
  auto load_state = [&](int ct) {
    const float* S_c = A.before + (((size_t)c * A.heads + h) * dv + ct * 16 + l16) * dk + 4 * g;
#pragma unroll
    for (int k = 0; k < KS; ++k) sb[k] = *(const floatx4*)(S_c + min(k * 16, dk - 16));
  };
  if ((wave >> 1) * 16 < dv) load_state(wave >> 1);
  __syncthreads();
  // P[i][j] = d^(i - j) (q_i . k_j) for j <= i: ten tiles of 16 x 16
  for (int tile = wave; tile < 10; tile += 8) {
    const int rt = tile >= 6 ? 3 : tile >= 3 ? 2 : tile >= 1 ? 1 : 0;
    const int ct = tile - rt * (rt + 1) / 2;
    const float* qa = Qs + (rt * 16 + l16) * QLD + 4 * g;
    const float* kb = Ks + (ct * 16 + l16) * QLD + 4 * g;
    floatx4 acc = {0.f, 0.f, 0.f, 0.f}, acc2 = {0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
    for (int k0 = 0; k0 < dk; k0 += 16) {
      const floatx4 a = *(const floatx4*)(qa + k0), b = *(const floatx4*)(kb + k0);
      acc = mfma_f32(a[0], b[0], acc);
      acc2 = mfma_f32(a[1], b[1], acc2);
      acc = mfma_f32(a[2], b[2], acc);
      acc2 = mfma_f32(a[3], b[3], acc2);
    }
    acc += acc2;
    const int j = ct * 16 + l16;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int i = rt * 16 + 4 * g + e;
      Ps[tile * LIN_PTILE + (4 * g + e) * LIN_PLD + l16] = j <= i ? acc[e] * pw[max(i - j, 0)] : 0.f;
    }
  }
  __syncthreads();  // K has been read: V takes its place
#pragma unroll
  for (int j = 0; j < NV; ++j)
    if (512 * j < LIN_ROWS * v4) {
      const int idx = tid + 512 * j;
      const int t = idx / v4;
      float v[4];
#pragma unroll
      for (int e = 0; e < 4; ++e) v[e] = t < have ? lin_act<T>(vr[j].get(e), A.silu) : 0.f;
      if (t < LIN_ROWS) *(float4*)(Ks + t * vld + idx % v4 * 4) = float4{v[0], v[1], v[2], v[3]};
    }
  __syncthreads();
  // a wave takes two row tiles (one early, one late: their causal parts add up to the same) of a tile of value columns
  const int rts[2] = {wave & 1, 3 - (wave & 1)};
  for (int ct = wave >> 1; ct * 16 < dv; ct += 4) {
    floatx4 acc[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};
#pragma unroll
    for (int k = 0; k < KS; ++k) {
      if (k * 16 >= dk) break;
      floatx4 a[2];
#pragma unroll
      for (int r = 0; r < 2; ++r) a[r] = *(const floatx4*)(Qs + (rts[r] * 16 + l16) * QLD + 4 * g + k * 16);
#pragma unroll
      for (int e = 0; e < 4; ++e)
#pragma unroll
        for (int r = 0; r < 2; ++r) acc[r] = mfma_f32(a[r][e], sb[k][e], acc[r]);
    }
    if ((ct + 4) * 16 < dv) load_state(ct + 4);
#pragma unroll
    for (int r = 0; r < 2; ++r) {
#pragma unroll
      for (int e = 0; e < 4; ++e) acc[r][e] *= pw[rts[r] * 16 + 4 * g + e + 1];
      const float* pa = Ps + rts[r] * (rts[r] + 1) / 2 * LIN_PTILE + l16 * LIN_PLD + 4 * g;
      for (int j = 0; j <= rts[r]; ++j) {
        const floatx4 a = *(const floatx4*)(pa + j * LIN_PTILE);
#pragma unroll
        for (int e = 0; e < 4; ++e) acc[r] = mfma_f32(a[e], Ks[(j * 16 + 4 * g + e) * vld + ct * 16 + l16], acc[r]);
      }
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int t = rts[r] * 16 + 4 * g + e;
        if (t < have) A.out[(size_t)(lo + t) * A.ldo + (size_t)h * dv + ct * 16 + l16] = acc[r][e];
      }
    }
  }
}

// ---------------------------------------------------------------------------------------------------------------------
// the chunked form with a channel decay

// the value of another lane of the row of 16: of the partner block of 1, 2, 4 or 8 lanes (of any of its lanes)
template <int S>
__device__ __forceinline__ float partner(float v) {
  constexpr int CTRL = S == 1 ? 0xB1 : S == 2 ? 0x4E : S == 4 ? 0x141 : 0x140;
  return __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), CTRL, 0xF, 0xF, true));
}

// Products of the alphas of a tile's 16 rows, of which a lane holds one (its place l16 in the row of lanes): up to and with
// the lane's own row (p), of the rows behind it (u), of all (t); over blocks of 1, 2, 4, 8, 16 rows as `widen` is called.
struct TileProducts {
  float p, u, t;
  __device__ __forceinline__ void start(float alpha) { p = alpha, u = 1.0f, t = alpha; }
  template <int S>
  __device__ __forceinline__ void widen(int l16) {  // from blocks of S rows to blocks of 2 S
    const float o = partner<S>(t);
    if (l16 & S)
      p *= o;
    else
      u *= o;
    t *= o;
  }
};

// z of a channel decay for 16 channels (from channel row `w` of W_up on) and 16 rows (a lane holds the one at `m`): lane l gets
// row l % 16, channels 4 (l / 16) .. + 4, which is how a product of [channels x middle] and [middle x rows] leaves them
template <typename T>
struct DecayInput;
template <>
struct DecayInput<bf16_t> {
  static __device__ __forceinline__ floatx4 make(const bf16_t* w, const bf16_t* m, int middle, int l16, int g, floatx4 z) {
    for (int k0 = 0; k0 < middle; k0 += LIN_MIDDLE) {
      const u32x4 a = *(const u32x4*)(w + (size_t)l16 * middle + k0 + 8 * g);
      const u32x4 b = *(const u32x4*)(m + k0 + 8 * g);
      z = mfma16(a, b, z);
    }
    return z;
  }
};
template <>
struct DecayInput<float> {
  static __device__ __forceinline__ floatx4 make(const float* w, const float* m, int middle, int l16, int g, floatx4 z) {
    for (int k0 = 0; k0 < middle; k0 += 16) {
      const floatx4 a = *(const floatx4*)(w + (size_t)l16 * middle + k0 + 4 * g);
      const floatx4 b = *(const floatx4*)(m + k0 + 4 * g);
#pragma unroll
      for (int e = 0; e < 4; ++e) z = mfma_f32(a[e], b[e], z);
    }
    return z;
  }
};

// A wave stages the rows of tile wave % 4 in every other group of 16 channels from wave / 4 on; lane l: row l % 16, channels
// 4 (l / 16) .. + 4 of the group.
// grid (chunk, head, 128 value columns), eight waves, as linear_local
template <typename T, int DT>
__global__ __launch_bounds__(512) void linear_channel_local_kernel(LinArgs A) {
  constexpr int DKP = DT * 64;
  constexpr int KLD = DKP + 16;
  constexpr int VLD = LIN_LOCAL_COLS + 16;
  constexpr int NB = DKP / 32;  // groups of 16 channels per wave
  __shared__ __align__(16) float Ks[LIN_ROWS * KLD];
  __shared__ __align__(16) float Vs[LIN_ROWS * VLD];
  __shared__ __align__(16) float Tot[4 * DKP];
  const int tid = threadIdx.x;
  const int wave = tid >> 6, lane = tid & 63, l16 = lane & 15, g = lane >> 4;
  const int c = blockIdx.x, h = blockIdx.y, col0 = blockIdx.z * LIN_LOCAL_COLS;
  const int lo = A.chunks[c * 2], have = A.chunks[c * 2 + 1];
  const int dk = A.dk, dv = A.dv;
  const int vcols = min(LIN_LOCAL_COLS, dv - col0);
  const T* y = (const T*)A.y;
  const T* vh = y + A.v_off + (size_t)h * dv + col0;
  const int rt = wave & 3, b0 = wave >> 2;
  const int row = rt * 16 + l16;
  const bool on = row < have;
  const size_t at = (size_t)(lo + min(row, have - 1));  // rows beyond the chunk's are read from its last one and dropped
  Raw4<T> ku[NB], vu[4];
  floatx4 zu[NB];
#pragma unroll
  for (int b = 0; b < NB; ++b) {
    const int i0 = min((b0 + 2 * b) * 16, dk - 16), i = i0 + 4 * g;
    ku[b].load(y + at * A.ld + A.k_off + (size_t)h * dk + i);
    zu[b] = DecayInput<T>::make((const T*)A.w_up + ((size_t)h * dk + i0) * A.middle, y + at * A.ld + A.m_off, A.middle, l16, g,
                                *(const floatx4*)(A.b_up + (size_t)h * dk + i));
  }
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    const int t = (tid >> 5) + 16 * j;
    vu[j].load(vh + (size_t)(lo + min(t, have - 1)) * A.ld + min((tid & 31) * 4, vcols - 4));
  }
  float u[NB][4];
#pragma unroll
  for (int b = 0; b < NB; ++b) {
    float tot[4];
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      TileProducts tp;
      tp.start(on ? channel_alpha<T>(zu[b][e], A.inv_tau) : 1.0f);
      tp.widen<1>(l16);
      tp.widen<2>(l16);
      tp.widen<4>(l16);
      tp.widen<8>(l16);
      u[b][e] = tp.u;
      tot[e] = tp.t;
    }
    if (l16 == 0) *(float4*)(Tot + rt * DKP + (b0 + 2 * b) * 16 + 4 * g) = float4{tot[0], tot[1], tot[2], tot[3]};
  }
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    const int t = (tid >> 5) + 16 * j;
    const bool von = t < have && (tid & 31) * 4 < vcols;
    float v[4];
#pragma unroll
    for (int e = 0; e < 4; ++e) v[e] = von ? lin_act<T>(vu[j].get(e), A.silu) : 0.f;
    *(float4*)(Vs + t * VLD + (tid & 31) * 4) = float4{v[0], v[1], v[2], v[3]};
  }
  __syncthreads();
#pragma unroll
  for (int b = 0; b < NB; ++b) {
    const int i = (b0 + 2 * b) * 16 + 4 * g;
    floatx4 w = {u[b][0], u[b][1], u[b][2], u[b][3]};
    for (int r = rt + 1; r < 4; ++r) w *= *(const floatx4*)(Tot + r * DKP + i);
    float k[4];
#pragma unroll
    for (int e = 0; e < 4; ++e) k[e] = on && i < dk ? lin_act<T>(ku[b].get(e), A.silu) * A.k_scale * w[e] : 0.f;
    *(float4*)(Ks + row * KLD + i) = float4{k[0], k[1], k[2], k[3]};
  }
  if (blockIdx.z == 0 && tid < dk)
    A.chunk_decay[((size_t)c * A.heads + h) * dk + tid] = (Tot[tid] * Tot[DKP + tid]) * (Tot[2 * DKP + tid] * Tot[3 * DKP + tid]);
  __syncthreads();
  const int dk_tile = (wave & 3) * DT, v_tile = (wave >> 2) * 4;
  if (dk_tile * 16 >= dk || v_tile * 16 >= vcols) return;  // nothing of this wave's is in the matrix
  floatx4 S[DT][4];
#pragma unroll
  for (int j = 0; j < DT; ++j)
#pragma unroll
    for (int n = 0; n < 4; ++n) S[j][n] = floatx4{0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
  for (int t0 = 0; t0 < have; t0 += 4) {
    float a[DT], b[4];
#pragma unroll
    for (int j = 0; j < DT; ++j) a[j] = Ks[(t0 + g) * KLD + (dk_tile + j) * 16 + l16];
#pragma unroll
    for (int n = 0; n < 4; ++n) b[n] = Vs[(t0 + g) * VLD + (v_tile + n) * 16 + l16];
#pragma unroll
    for (int n = 0; n < 4; ++n)
      if ((v_tile + n) * 16 < vcols) {
#pragma unroll
        for (int j = 0; j < DT; ++j) S[j][n] = mfma_f32(a[j], b[n], S[j][n]);
      }
  }
#pragma unroll
  for (int j = 0; j < DT; ++j) {
    const int i = (dk_tile + j) * 16 + 4 * g;
    if (i >= dk) continue;
#pragma unroll
    for (int n = 0; n < 4; ++n)
      if ((v_tile + n) * 16 < vcols)
        *(floatx4*)(A.before + (((size_t)c * A.heads + h) * dv + col0 + (v_tile + n) * 16 + l16) * dk + i) = S[j][n];
  }
}

// the pairs of level S (i > j, highest differing bit S) of a tile: the product of the second halves' rows, each times the
// alphas of its half up to it, with the first halves' rows, each times the alphas of its half behind it; accumulated over
// four channels
template <int S>
__device__ __forceinline__ void level_product(const float (&q)[4], const float (&k)[4], TileProducts (&tp)[4], int l16, floatx4& acc) {
#pragma unroll
  for (int e = 0; e < 4; ++e) {
    const bool second = l16 & S;
    acc = mfma_f32(second ? q[e] * tp[e].p : 0.f, second ? 0.f : k[e] * tp[e].u, acc);
    tp[e].widen<S>(l16);
  }
}

// grid (chunk, head), eight waves. LDS: Q [64][dk], the ten tiles of P on and below the diagonal, the tiles' products
// [4][dk], K [64][dk] (later V [64][dv] in its place).
template <typename T, int DT>
__global__ __launch_bounds__(512) void linear_channel_outputs_kernel(LinArgs A) {
  constexpr int DKP = DT * 64;
  constexpr int QLD = DKP + 4;
  constexpr int NB = DKP / 32;
  constexpr int NV = 8;  // pieces of V per thread, for values of up to 256
  constexpr int KS = DKP / 16;
  extern __shared__ __align__(16) float lin_smem[];
  float* Qs = lin_smem;
  float* Ps = Qs + LIN_ROWS * QLD;
  float* Tot = Ps + 10 * 256;
  float* Ks = Tot + 4 * DKP;
  const int tid = threadIdx.x;
  const int wave = tid >> 6, lane = tid & 63, l16 = lane & 15, g = lane >> 4;
  const int c = blockIdx.x, h = blockIdx.y;
  const int lo = A.chunks[c * 2], have = A.chunks[c * 2 + 1];
  const int dk = A.dk, dv = A.dv, vld = dv + 4, v4 = dv >> 2;
  const T* y = (const T*)A.y;
  const int rt = wave & 3, b0 = wave >> 2;
  const int row = rt * 16 + l16;
  const bool on = row < have;
  float qh[NB][4];  // this lane's row: q times the alphas of the tile up to the row
  floatx4 dg;       // the tile's pairs, this wave's channels
  {
    const size_t at = (size_t)(lo + min(row, have - 1));
    Raw4<T> qu[NB], ku[NB];
    floatx4 zu[NB];
#pragma unroll
    for (int b = 0; b < NB; ++b) {
      const int i0 = min((b0 + 2 * b) * 16, dk - 16), i = i0 + 4 * g;
      qu[b].load(y + at * A.ld + A.q_off + (size_t)h * dk + i);
      ku[b].load(y + at * A.ld + A.k_off + (size_t)h * dk + i);
      zu[b] = DecayInput<T>::make((const T*)A.w_up + ((size_t)h * dk + i0) * A.middle, y + at * A.ld + A.m_off, A.middle, l16, g,
                                  *(const floatx4*)(A.b_up + (size_t)h * dk + i));
    }
    floatx4 acc1 = {0.f, 0.f, 0.f, 0.f}, acc2 = acc1, acc4 = acc1, acc8 = acc1;
    float own = 0.f;  // q_i . k_i
#pragma unroll
    for (int b = 0; b < NB; ++b) {
      const int i = (b0 + 2 * b) * 16 + 4 * g;
      const bool in = on && i < dk;
      float q[4], k[4];
      TileProducts tp[4];
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        q[e] = in ? lin_act<T>(qu[b].get(e), A.silu) : 0.f;
        k[e] = in ? lin_act<T>(ku[b].get(e), A.silu) * A.k_scale : 0.f;
        own = fmaf(q[e], k[e], own);
        tp[e].start(on ? channel_alpha<T>(zu[b][e], A.inv_tau) : 1.0f);
      }
      level_product<1>(q, k, tp, l16, acc1);
      level_product<2>(q, k, tp, l16, acc2);
      level_product<4>(q, k, tp, l16, acc4);
      level_product<8>(q, k, tp, l16, acc8);
#pragma unroll
      for (int e = 0; e < 4; ++e) qh[b][e] = q[e] * tp[e].p;
      if (i < dk) {
        *(float4*)(Qs + row * QLD + i) = float4{qh[b][0], qh[b][1], qh[b][2], qh[b][3]};
        *(float4*)(Ks + row * QLD + i) = float4{k[0] * tp[0].u, k[1] * tp[1].u, k[2] * tp[2].u, k[3] * tp[3].u};
        if (l16 == 0) *(float4*)(Tot + rt * DKP + i) = float4{tp[0].t, tp[1].t, tp[2].t, tp[3].t};
      }
    }
    own += __shfl_xor(own, 16, 64);
    own += __shfl_xor(own, 32, 64);
#pragma unroll
    for (int e = 0; e < 4; ++e) {  // place (i, j) = (4 g + e, l16)
      const int i = 4 * g + e, x = i ^ l16;
      const float v = x >= 8 ? acc8[e] : x >= 4 ? acc4[e] : x >= 2 ? acc2[e] : x >= 1 ? acc1[e] : own;
      dg[e] = i >= l16 ? v : 0.f;
      if (b0 == 0) Ps[(rt * (rt + 3) / 2) * 256 + i * 16 + l16] = dg[e];
    }
  }
  Raw4<T> vr[NV];  // in flight while P is computed
#pragma unroll
  for (int j = 0; j < NV; ++j)
    if (512 * j < LIN_ROWS * v4) {
      const int idx = tid + 512 * j;
      vr[j].load(y + (size_t)(lo + min(idx / v4, have - 1)) * A.ld + A.v_off + (size_t)h * dv + idx % v4 * 4);
    }
  // the state's part for this wave's first tile of value columns, in flight too; entries beyond dk are read from the last
  floatx4 sb[KS];
  auto load_state = [&](int ct) {
    const float* S_c = A.before + (((size_t)c * A.heads + h) * dv + ct * 16 + l16) * dk + 4 * g;
#pragma unroll
    for (int k = 0; k < KS; ++k) sb[k] = *(const floatx4*)(S_c + min(k * 16, dk - 16));
  };
  if ((wave >> 1) * 16 < dv) load_state(wave >> 1);
  __syncthreads();
  if (b0 == 1) {  // the other half of the channels
#pragma unroll
    for (int e = 0; e < 4; ++e) Ps[(rt * (rt + 3) / 2) * 256 + (4 * g + e) * 16 + l16] += dg[e];
  }
  // the six tiles below the diagonal: waves 0 .. 5
  if (wave < 6) {
    const int r = wave < 1 ? 1 : wave < 3 ? 2 : 3, ct = wave - r * (r - 1) / 2;
    const float* qa = Qs + (r * 16 + l16) * QLD + 4 * g;
    const float* kb = Ks + (ct * 16 + l16) * QLD + 4 * g;
    floatx4 acc = {0.f, 0.f, 0.f, 0.f}, acc2 = {0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
    for (int k0 = 0; k0 < dk; k0 += 16) {
      floatx4 a = *(const floatx4*)(qa + k0);
      const floatx4 b = *(const floatx4*)(kb + k0);
      for (int m = ct + 1; m < r; ++m) a *= *(const floatx4*)(Tot + m * DKP + k0 + 4 * g);
      acc = mfma_f32(a[0], b[0], acc);
      acc2 = mfma_f32(a[1], b[1], acc2);
      acc = mfma_f32(a[2], b[2], acc);
      acc2 = mfma_f32(a[3], b[3], acc2);
    }
    acc += acc2;
#pragma unroll
    for (int e = 0; e < 4; ++e) Ps[(r * (r + 1) / 2 + ct) * 256 + (4 * g + e) * 16 + l16] = acc[e];
  }
  __syncthreads();  // Q and K have been read: V takes K's place, Q gets the alphas of the tiles before
#pragma unroll
  for (int b = 0; b < NB; ++b) {
    const int i = (b0 + 2 * b) * 16 + 4 * g;
    if (i >= dk) continue;
    floatx4 w = {qh[b][0], qh[b][1], qh[b][2], qh[b][3]};
    for (int m = 0; m < rt; ++m) w *= *(const floatx4*)(Tot + m * DKP + i);
    *(floatx4*)(Qs + row * QLD + i) = w;
  }
#pragma unroll
  for (int j = 0; j < NV; ++j)
    if (512 * j < LIN_ROWS * v4) {
      const int idx = tid + 512 * j;
      const int t = idx / v4;
      float v[4];
#pragma unroll
      for (int e = 0; e < 4; ++e) v[e] = t < have ? lin_act<T>(vr[j].get(e), A.silu) : 0.f;
      if (t < LIN_ROWS) *(float4*)(Ks + t * vld + idx % v4 * 4) = float4{v[0], v[1], v[2], v[3]};
    }
  __syncthreads();
  // a wave takes two row tiles (one early, one late: their causal parts add up to the same) of a tile of value columns
  const int rts[2] = {wave & 1, 3 - (wave & 1)};
  for (int ct = wave >> 1; ct * 16 < dv; ct += 4) {
    floatx4 acc[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};
#pragma unroll
    for (int k = 0; k < KS; ++k) {
      if (k * 16 >= dk) break;
      floatx4 a[2];
#pragma unroll
      for (int r = 0; r < 2; ++r) a[r] = *(const floatx4*)(Qs + (rts[r] * 16 + l16) * QLD + 4 * g + k * 16);
#pragma unroll
      for (int e = 0; e < 4; ++e)
#pragma unroll
        for (int r = 0; r < 2; ++r) acc[r] = mfma_f32(a[r][e], sb[k][e], acc[r]);
    }
    if ((ct + 4) * 16 < dv) load_state(ct + 4);
#pragma unroll
    for (int r = 0; r < 2; ++r) {
      const float* pa = Ps + rts[r] * (rts[r] + 1) / 2 * 256 + l16 * 16 + 4 * g;
      for (int j = 0; j <= rts[r]; ++j) {
        const floatx4 a = *(const floatx4*)(pa + j * 256);
#pragma unroll
        for (int e = 0; e < 4; ++e) acc[r] = mfma_f32(a[e], Ks[(j * 16 + 4 * g + e) * vld + ct * 16 + l16], acc[r]);
      }
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int t = rts[r] * 16 + 4 * g + e;
        if (t < have) A.out[(size_t)(lo + t) * A.ldo + (size_t)h * dv + ct * 16 + l16] = acc[r][e];
      }
    }
  }
}

template <typename T, int DT>
static int launch_channel_outputs(dim3 grid, hipStream_t stream, const LinArgs& A) {
  const int qld = DT * 64 + 4, vld = A.dv + 4;
  const size_t smem = ((size_t)LIN_ROWS * (qld + (qld > vld ? qld : vld)) + 10 * 256 + 4 * DT * 64) * sizeof(float);
  static size_t raised = 64 * 1024;
  if (smem > raised) {
    if (smem > 160 * 1024 ||
        hipFuncSetAttribute((const void*)linear_channel_outputs_kernel<T, DT>, hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024) != hipSuccess)
      return -1;
    raised = 160 * 1024;
  }
  linear_channel_outputs_kernel<T, DT><<<grid, 512, smem, stream>>>(A);
  return 0;
}

template <typename T, int DT, bool ROT>
static int launch_outputs(dim3 grid, hipStream_t stream, const LinArgs& A) {
  const int qld = DT * 64 + 4, vld = A.dv + 4;
  const size_t smem = ((size_t)LIN_ROWS * (qld + (qld > vld ? qld : vld)) + 10 * LIN_PTILE) * sizeof(float);
  static size_t raised = 64 * 1024;
  if (smem > raised) {
    if (smem > 160 * 1024 ||
        hipFuncSetAttribute((const void*)linear_outputs_kernel<T, DT, ROT>, hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024) != hipSuccess)
      return -1;
    raised = 160 * 1024;
  }
  linear_outputs_kernel<T, DT, ROT><<<grid, 512, smem, stream>>>(A);
  return 0;
}

static int check_args(const char* name, const LinArgs& A, int n_requests) {
  if (A.heads <= 0 || A.heads > 65535 || A.dk <= 0 || A.dk > LIN_PARTS * 16 || A.dv <= 0 || A.dv > LIN_COLS * 65535)
    JLLM_FAIL("%s: %d heads, key size %d (1..%d are taken), value size %d", name, A.heads, A.dk, LIN_PARTS * 16, A.dv);
  if (n_requests <= 0 || n_requests > A.n_rows) JLLM_FAIL("%s: %d requests in %d rows", name, n_requests, A.n_rows);
  if (A.q_off < 0 || A.k_off < 0 || A.v_off < 0 || A.ld < A.q_off + A.heads * A.dk || A.ld < A.k_off + A.heads * A.dk ||
      A.ld < A.v_off + A.heads * A.dv || A.ldo < A.heads * A.dv)
    JLLM_FAIL("%s: short rows", name);
  if (A.rot < 0 || A.rot % 2 || A.rot > A.dk || (A.rot && (!A.cos_t || !A.sin_t || !A.positions)))
    JLLM_FAIL("%s: a rotary width of %d for heads of %d", name, A.rot, A.dk);
  if ((A.w_up == nullptr) == (A.powers == nullptr)) JLLM_FAIL("%s: a decay per head or per channel", name);
  if (A.w_up && (!A.b_up || A.middle <= 0 || A.middle % LIN_MIDDLE || A.rank <= 0 || A.rank > A.middle || A.m_off < 0 || A.ld < A.m_off + A.middle || !(A.inv_tau > 0.f) || A.rot))
    JLLM_FAIL("%s: a channel decay from columns %d .. + %d of rows of %d (1 / tau %g, rotary width %d)", name, A.m_off, A.middle, A.ld, (double)A.inv_tau, A.rot);
  return 0;
}

extern "C" int jllm_linear_scan(const void* y, int ld, int q_off, int k_off, int v_off, int dtype, const int* positions,
                                const float* cos_t, const float* sin_t, int rot, int silu, float k_scale, const float* powers,
                                float* state, float* out, int ldo, const int* row_req, const int* state_slots, int n_rows,
                                int n_requests, int heads, int dk, int dv, int m_off, int middle, int rank, const void* w_up,
                                const float* b_up, float inv_tau, hipStream_t stream) {
  if (n_rows <= 0) return 0;
  LinArgs A{y, ld, q_off, k_off, v_off, positions, cos_t, sin_t, rot, silu, k_scale, powers, state, out, ldo, row_req, state_slots,
            n_rows, heads, dk, dv, nullptr, nullptr, nullptr, m_off, middle, rank, w_up, b_up, inv_tau, nullptr};
  if (check_args("linear_scan", A, n_requests) != 0) return -1;
  dim3 grid(n_requests, heads, (dv + LIN_COLS - 1) / LIN_COLS);
  const int per_lane = (dk + LIN_PARTS - 1) / LIN_PARTS;
  const bool few = n_rows <= 2 * n_requests;
#define LIN_LAUNCH(E)                                                             \
  do {                                                                            \
    if (w_up && few)                                                              \
      linear_scan_kernel<T, E, 2, false, true><<<grid, 256, 0, stream>>>(A);      \
    else if (w_up)                                                                \
      linear_scan_kernel<T, E, 16, false, true><<<grid, 256, 0, stream>>>(A);     \
    else if (few && rot)                                                          \
      linear_scan_kernel<T, E, 2, true, false><<<grid, 256, 0, stream>>>(A);      \
    else if (few)                                                                 \
      linear_scan_kernel<T, E, 2, false, false><<<grid, 256, 0, stream>>>(A);     \
    else if (rot)                                                                 \
      linear_scan_kernel<T, E, 16, true, false><<<grid, 256, 0, stream>>>(A);     \
    else                                                                          \
      linear_scan_kernel<T, E, 16, false, false><<<grid, 256, 0, stream>>>(A);    \
  } while (0)
  JLLM_DISPATCH_1(dtype, T, {
    if (per_lane <= 2)
      LIN_LAUNCH(2);
    else if (per_lane <= 4)
      LIN_LAUNCH(4);
    else if (per_lane <= 8)
      LIN_LAUNCH(8);
    else
      LIN_LAUNCH(16);
  })
#undef LIN_LAUNCH
  JLLM_CHECK_LAUNCH("linear_scan");
  return 0;
}

// Returns 1 (declined) for sizes that the chunked form does not take. requests [n_requests, 3]: first row, rows, first
// chunk; chunks [n_chunks, 2]: first row, rows (at most 64, of one request, in order); before: fp32 [n_chunks, heads, dv, dk];
// with w_up (a channel decay, powers null) chunk_decay: fp32 [n_chunks, heads, dk]
extern "C" int jllm_linear_chunks(const void* y, int ld, int q_off, int k_off, int v_off, int dtype, const int* positions,
                                  const float* cos_t, const float* sin_t, int rot, int silu, float k_scale,
                                  const float* powers, float* state, float* out, int ldo, const int* requests,
                                  const int* chunks, int n_chunks, float* before, const int* state_slots, int n_rows,
                                  int n_requests, int heads, int dk, int dv, int m_off, int middle, int rank, const void* w_up,
                                  const float* b_up, float inv_tau, float* chunk_decay, hipStream_t stream) {
  if (n_rows <= 0) return 0;
  LinArgs A{y, ld, q_off, k_off, v_off, positions, cos_t, sin_t, rot, silu, k_scale, powers, state, out, ldo, nullptr, state_slots,
            n_rows, heads, dk, dv, requests, chunks, before, m_off, middle, rank, w_up, b_up, inv_tau, chunk_decay};
  if (check_args("linear_chunks", A, n_requests) != 0) return -1;
  if (n_chunks < n_requests || n_chunks > n_rows || !requests || !chunks || !before) JLLM_FAIL("linear_chunks: %d chunks of %d rows of %d requests", n_chunks, n_rows, n_requests);
  const size_t bytes4 = dtype == JLLM_F32 ? 16 : 8;
  if ((dk & 15) || (dv & 15) || dk > 256 || dv > 256 || (rot & 7)) return 1;
  if ((ld & 3) || (q_off & 3) || (k_off & 3) || (v_off & 3) || ((uintptr_t)y % bytes4) || ((uintptr_t)state & 15) || ((uintptr_t)before & 15) ||
      (rot && (((uintptr_t)cos_t & 15) || ((uintptr_t)sin_t & 15))))
    return 1;
  if (n_requests > 65535) return 1;
  const int per16 = dtype == JLLM_F32 ? 4 : 8;  // elements in 16 bytes
  if (w_up && (ld % per16 || m_off % per16 || ((uintptr_t)y & 15) || ((uintptr_t)w_up & 15) || ((uintptr_t)b_up & 15) || ((uintptr_t)chunk_decay & 15)))
    return 1;
  if (w_up && !chunk_decay) JLLM_FAIL("linear_chunks: no place for the chunks' decays");
  const dim3 lgrid(n_chunks, heads, (dv + LIN_LOCAL_COLS - 1) / LIN_LOCAL_COLS), cgrid((unsigned)(((size_t)dk * dv / 4 + 255) / 256), heads, n_requests), ogrid(n_chunks, heads);
  int rc = 0;
#define LIN_CHUNKS(DT)                                                                     \
  do {                                                                                     \
    if (w_up) {                                                                            \
      linear_channel_local_kernel<T, DT><<<lgrid, 512, 0, stream>>>(A);                    \
      linear_combine_kernel<true><<<cgrid, 256, 0, stream>>>(A);                           \
      rc = launch_channel_outputs<T, DT>(ogrid, stream, A);                                \
      break;                                                                               \
    }                                                                                      \
    if (rot)                                                                               \
      linear_local_kernel<T, DT, true><<<lgrid, 512, 0, stream>>>(A);                      \
    else                                                                                   \
      linear_local_kernel<T, DT, false><<<lgrid, 512, 0, stream>>>(A);                     \
    linear_combine_kernel<false><<<cgrid, 256, 0, stream>>>(A);                            \
    rc = rot ? launch_outputs<T, DT, true>(ogrid, stream, A) : launch_outputs<T, DT, false>(ogrid, stream, A); \
  } while (0)
  JLLM_DISPATCH_1(dtype, T, {
    if (dk <= 64)
      LIN_CHUNKS(1);
    else if (dk <= 128)
      LIN_CHUNKS(2);
    else
      LIN_CHUNKS(4);
  })
#undef LIN_CHUNKS
  if (rc < 0) JLLM_FAIL("linear_chunks: cannot reserve LDS");
  JLLM_CHECK_LAUNCH("linear_chunks");
  return 0;
}
