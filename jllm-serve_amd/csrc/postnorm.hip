// What lies between two sublayers when a norm sits on a sublayer's output, and the mix of a row with the previous token's
// row.
//
//   rms_between   for sublayers that are normed on both sides. Per row, each part optional: t = s1 a (+ s2 a2) and x +=
//                 rms(t) g; x += the row's further row (the embedding output); x += a vector; and the norm of the new row
//                 for the next sublayer's products, rms(x) g'.
//   rms_seam      per row: t = a, or, for two branches side by side, t = s1 rms(a) w1 + s2 rms(a2) w2; the residual row
//                 x += rms(t) g; and the new row for the next reader: as it is, or shifted, x + (x' - x) mu with x' the
//                 request's previous row. The shifted form is for steps in which every request brings one row: x' is
//                 then the request's state, which becomes the new x in the same launch.
//   token_shift   out = h + (h' - h) mu for rows of any step, h' the row before of the same request (its state for the
//                 first row of the step, zeros at position 0: a fresh request's state is zero); for steps of single rows
//                 it advances the state in the same launch, otherwise token_shift_advance does.
// rms(v) = v / sqrt(mean(v^2) + eps). The residual, the state, every vector and all sums are fp32.
#include <math.h>

#include "common.h"

#define PN_THREADS 256

__device__ __forceinline__ float pn_block_sum(float v, float* red) {  // red: PN_THREADS / 64 floats of this sum's own
  v = wave_sum(v);
  if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
  __syncthreads();
  float s = 0.f;
#pragma unroll
  for (int i = 0; i < PN_THREADS / 64; ++i) s += red[i];
  return s;
}

// V neighbouring elements (4, or 1 where the rows do not allow it)
template <int V>
__device__ __forceinline__ void pn_load(const float* p, float (&v)[V]) {
  if constexpr (V == 4) {
    const float4 t = *(const float4*)p;
    v[0] = t.x, v[1] = t.y, v[2] = t.z, v[3] = t.w;
  } else {
    v[0] = p[0];
  }
}
template <int V>
__device__ __forceinline__ void pn_load(const bf16_t* p, float (&v)[V]) {
  if constexpr (V == 4) {
    const uint2 t = *(const uint2*)p;
    v[0] = __uint_as_float(t.x << 16), v[1] = __uint_as_float(t.x & 0xffff0000u);
    v[2] = __uint_as_float(t.y << 16), v[3] = __uint_as_float(t.y & 0xffff0000u);
  } else {
    v[0] = bf16_to_f32(p[0]);
  }
}
template <int V>
__device__ __forceinline__ void pn_store(float* p, const float (&v)[V]) {
  if constexpr (V == 4)
    *(float4*)p = float4{v[0], v[1], v[2], v[3]};
  else
    p[0] = v[0];
}
template <int V>
__device__ __forceinline__ void pn_store(bf16_t* p, const float (&v)[V]) {
  if constexpr (V == 4) {
    uint2 t;
    t.x = (uint32_t)f32_to_bf16(v[0]).bits | ((uint32_t)f32_to_bf16(v[1]).bits << 16);
    t.y = (uint32_t)f32_to_bf16(v[2]).bits | ((uint32_t)f32_to_bf16(v[3]).bits << 16);
    *(uint2*)p = t;
  } else {
    p[0] = f32_to_bf16(v[0]);
  }
}

struct SeamArgs {
  float* x;  // [rows, d]
  int d;
  const void* a;  // [rows, lda]
  int lda;
  const void* a2;  // or null
  int lda2;
  float s1, s2;
  const float* w1;  // the branches' gains, with a2
  const float* w2;
  float branch_eps;
  const float* gain;
  float eps;
  void* out;  // [rows, ldo] or null
  int ldo;
  const float* mu;  // or null: the row as it is
  float* state;     // [slots, d]
  const int* state_slots;
};

template <typename TA, typename TO, int V, int G>
__global__ __launch_bounds__(PN_THREADS) void rms_seam_kernel(SeamArgs A) {
  __shared__ float red[3 * (PN_THREADS / 64)];
  const int r = blockIdx.x, d = A.d;
  float* xr = A.x + (size_t)r * d;
  const TA* a = (const TA*)A.a + (size_t)r * A.lda;
  const bool two = A.a2 != nullptr;
  const TA* a2 = two ? (const TA*)A.a2 + (size_t)r * A.lda2 : a;
  float* st = A.mu ? A.state + (size_t)A.state_slots[r] * d : nullptr;
  // everything the row needs is requested before the first sum
  float x[G][V], t[G][V], u[G][V], gn[G][V], w1[G][V], w2[G][V], mu[G][V], pv[G][V];
#pragma unroll
  for (int k = 0; k < G; ++k) {
    const int i = (threadIdx.x + k * PN_THREADS) * V;
#pragma unroll
    for (int e = 0; e < V; ++e) x[k][e] = t[k][e] = u[k][e] = gn[k][e] = w1[k][e] = w2[k][e] = mu[k][e] = pv[k][e] = 0.f;
    if (i >= d) continue;
    pn_load<V>(xr + i, x[k]);
    pn_load<V>(a + i, t[k]);
    pn_load<V>(A.gain + i, gn[k]);
    if (two) {
      pn_load<V>(a2 + i, u[k]);
      pn_load<V>(A.w1 + i, w1[k]);
      pn_load<V>(A.w2 + i, w2[k]);
    }
    if (st) {
      pn_load<V>(A.mu + i, mu[k]);
      pn_load<V>(st + i, pv[k]);
    }
  }
  if (two) {
    float q1 = 0.f, q2 = 0.f;
#pragma unroll
    for (int k = 0; k < G; ++k)
#pragma unroll
      for (int e = 0; e < V; ++e) {
        q1 = fmaf(t[k][e], t[k][e], q1);
        q2 = fmaf(u[k][e], u[k][e], q2);
      }
    const float r1 = A.s1 * norm_scale(pn_block_sum(q1, red), d, A.branch_eps);
    const float r2 = A.s2 * norm_scale(pn_block_sum(q2, red + PN_THREADS / 64), d, A.branch_eps);
#pragma unroll
    for (int k = 0; k < G; ++k)
#pragma unroll
      for (int e = 0; e < V; ++e) t[k][e] = t[k][e] * r1 * w1[k][e] + u[k][e] * r2 * w2[k][e];
  }
  float q = 0.f;
#pragma unroll
  for (int k = 0; k < G; ++k)
#pragma unroll
    for (int e = 0; e < V; ++e) q = fmaf(t[k][e], t[k][e], q);
  const float rs = norm_scale(pn_block_sum(q, red + 2 * (PN_THREADS / 64)), d, A.eps);
#pragma unroll
  for (int k = 0; k < G; ++k) {
    const int i = (threadIdx.x + k * PN_THREADS) * V;
    if (i >= d) continue;
#pragma unroll
    for (int e = 0; e < V; ++e) x[k][e] += t[k][e] * rs * gn[k][e];
    pn_store<V>(xr + i, x[k]);
    if (!A.out) continue;
    float o[V];
#pragma unroll
    for (int e = 0; e < V; ++e) o[e] = st ? x[k][e] + (pv[k][e] - x[k][e]) * mu[k][e] : x[k][e];
    pn_store<V>((TO*)A.out + (size_t)r * A.ldo + i, o);
    if (st) pn_store<V>(st + i, x[k]);
  }
}

static bool pn_aligned(const void* p, size_t bytes) { return ((uintptr_t)p % bytes) == 0; }

struct BetweenArgs {
  float* x;  // [rows, d]
  int d;
  const void* a;  // [rows, lda] or null
  int lda;
  const void* a2;  // or null
  int lda2;
  float s1, s2;
  const float* gain;  // with a
  float eps;
  const float* rows;  // [rows, d] or null
  const void* vec;    // [d] or null
  int vec_bf16;
  const float* gain_next;  // with out
  float eps_next;
  void* out;  // [rows, ldo] or null
  int ldo;
};

template <typename TA, typename TO, int V, int G>
__global__ __launch_bounds__(PN_THREADS) void rms_between_kernel(BetweenArgs A) {
  __shared__ float red[2 * (PN_THREADS / 64)];
  const int r = blockIdx.x, d = A.d;
  float* xr = A.x + (size_t)r * d;
  const TA* a = A.a ? (const TA*)A.a + (size_t)r * A.lda : nullptr;
  const TA* a2 = A.a2 ? (const TA*)A.a2 + (size_t)r * A.lda2 : nullptr;
  // everything the row needs is requested before the first sum
  float x[G][V], t[G][V], u[G][V], gn[G][V], more[G][V], vec[G][V], nx[G][V];
#pragma unroll
  for (int k = 0; k < G; ++k) {
    const int i = (threadIdx.x + k * PN_THREADS) * V;
#pragma unroll
    for (int e = 0; e < V; ++e) x[k][e] = t[k][e] = u[k][e] = gn[k][e] = more[k][e] = vec[k][e] = nx[k][e] = 0.f;
    if (i >= d) continue;
    pn_load<V>(xr + i, x[k]);
    if (a) {
      pn_load<V>(a + i, t[k]);
      pn_load<V>(A.gain + i, gn[k]);
      if (a2) pn_load<V>(a2 + i, u[k]);
    }
    if (A.rows) pn_load<V>(A.rows + (size_t)r * d + i, more[k]);
    if (A.vec) {
      if (A.vec_bf16)
        pn_load<V>((const bf16_t*)A.vec + i, vec[k]);
      else
        pn_load<V>((const float*)A.vec + i, vec[k]);
    }
    if (A.out) pn_load<V>(A.gain_next + i, nx[k]);
  }
  if (a) {
    float q = 0.f;
#pragma unroll
    for (int k = 0; k < G; ++k)
#pragma unroll
      for (int e = 0; e < V; ++e) {
        t[k][e] = a2 ? fmaf(A.s2, u[k][e], A.s1 * t[k][e]) : A.s1 * t[k][e];
        q = fmaf(t[k][e], t[k][e], q);
      }
    const float rs = norm_scale(pn_block_sum(q, red), d, A.eps);
#pragma unroll
    for (int k = 0; k < G; ++k)
#pragma unroll
      for (int e = 0; e < V; ++e) x[k][e] += t[k][e] * rs * gn[k][e];
  }
  float q = 0.f;
#pragma unroll
  for (int k = 0; k < G; ++k) {
    const int i = (threadIdx.x + k * PN_THREADS) * V;
#pragma unroll
    for (int e = 0; e < V; ++e) {
      x[k][e] = (x[k][e] + more[k][e]) + vec[k][e];
      q = fmaf(x[k][e], x[k][e], q);
    }
    if (i < d && (a || A.rows || A.vec)) pn_store<V>(xr + i, x[k]);
  }
  if (!A.out) return;
  const float rs = norm_scale(pn_block_sum(q, red + PN_THREADS / 64), d, A.eps_next);
#pragma unroll
  for (int k = 0; k < G; ++k) {
    const int i = (threadIdx.x + k * PN_THREADS) * V;
    if (i >= d) continue;
    float o[V];
#pragma unroll
    for (int e = 0; e < V; ++e) o[e] = x[k][e] * rs * nx[k][e];
    pn_store<V>((TO*)A.out + (size_t)r * A.ldo + i, o);
  }
}

// a, a2 in a_dtype, the vector in vec_dtype; gains and rows fp32
extern "C" int jllm_rms_between(float* x, int n, int d, const void* a, int lda, const void* a2, int lda2, int a_dtype, float s1,
                                float s2, const float* gain, float eps, const float* rows, const void* vec, int vec_dtype,
                                const float* gain_next, float eps_next, void* out, int ldo, int out_dtype, hipStream_t stream) {
  if (n <= 0) return 0;
  if (d <= 0 || d > PN_THREADS * 32) JLLM_FAIL("rms_between: rows of %d entries (1..%d are taken)", d, PN_THREADS * 32);
  if (!x || (a && (!gain || lda < d)) || (a2 && (!a || lda2 < d))) JLLM_FAIL("rms_between: a branch without its gain or with short rows");
  if (out && (!gain_next || ldo < d)) JLLM_FAIL("rms_between: an output without its gain or with short rows");
  if (vec && vec_dtype != JLLM_F32 && vec_dtype != JLLM_BF16) JLLM_FAIL("rms_between: unknown dtype code %d", vec_dtype);
  BetweenArgs A{x, d, a, lda, a2, lda2, s1, s2, gain, eps, rows, vec, vec_dtype == JLLM_BF16, gain_next, eps_next, out, ldo};
  const size_t ea = a_dtype == JLLM_F32 ? 16 : 8, eo = out_dtype == JLLM_F32 ? 16 : 8, ev = vec_dtype == JLLM_F32 ? 16 : 8;
  const bool wide = d % 4 == 0 && pn_aligned(x, 16) && (!a || (pn_aligned(a, ea) && lda % 4 == 0 && pn_aligned(gain, 16))) &&
                    (!a2 || (pn_aligned(a2, ea) && lda2 % 4 == 0)) && pn_aligned(rows, 16) && (!vec || pn_aligned(vec, ev)) &&
                    (!out || (pn_aligned(out, eo) && ldo % 4 == 0 && pn_aligned(gain_next, 16)));
#define PN_LAUNCH(V, G) rms_between_kernel<TA, TO, V, G><<<n, PN_THREADS, 0, stream>>>(A)
  JLLM_DISPATCH_1(a_dtype, TA, {
    JLLM_DISPATCH_1(out_dtype, TO, {
      if (wide && d <= PN_THREADS * 4)
        PN_LAUNCH(4, 1);
      else if (wide && d <= PN_THREADS * 8)
        PN_LAUNCH(4, 2);
      else if (wide && d <= PN_THREADS * 16)
        PN_LAUNCH(4, 4);
      else if (wide)
        PN_LAUNCH(4, 8);
      else if (d <= PN_THREADS * 4)
        PN_LAUNCH(1, 4);
      else if (d <= PN_THREADS * 16)
        PN_LAUNCH(1, 16);
      else
        PN_LAUNCH(1, 32);
    })
  })
#undef PN_LAUNCH
  JLLM_CHECK_LAUNCH("rms_between");
  return 0;
}

// a, a2 in a_dtype; gains, mu and state fp32. mu: with `state` [slots, d] and the rows' slots, one row per request
extern "C" int jllm_rms_seam(float* x, int n, int d, const void* a, int lda, const void* a2, int lda2, int a_dtype, float s1,
                             float s2, const float* w1, const float* w2, float branch_eps, const float* gain, float eps,
                             void* out, int ldo, int out_dtype, const float* mu, float* state, const int* state_slots,
                             hipStream_t stream) {
  if (n <= 0) return 0;
  if (d <= 0 || d > PN_THREADS * 32) JLLM_FAIL("rms_seam: rows of %d entries (1..%d are taken)", d, PN_THREADS * 32);
  if (!x || !a || !gain || lda < d || (a2 && (lda2 < d || !w1 || !w2))) JLLM_FAIL("rms_seam: a branch without its gain or with short rows");
  if (out && ldo < d) JLLM_FAIL("rms_seam: short output rows");
  if (mu && (!out || !state || !state_slots)) JLLM_FAIL("rms_seam: a shift without its output or state");
  SeamArgs A{x, d, a, lda, a2, lda2, s1, s2, w1, w2, branch_eps, gain, eps, out, ldo, mu, state, state_slots};
  const size_t ea = a_dtype == JLLM_F32 ? 16 : 8, eo = out_dtype == JLLM_F32 ? 16 : 8;
  const bool wide = d % 4 == 0 && pn_aligned(x, 16) && pn_aligned(a, ea) && lda % 4 == 0 && pn_aligned(gain, 16) &&
                    (!a2 || (pn_aligned(a2, ea) && lda2 % 4 == 0 && pn_aligned(w1, 16) && pn_aligned(w2, 16))) &&
                    (!out || (pn_aligned(out, eo) && ldo % 4 == 0)) && (!mu || (pn_aligned(mu, 16) && pn_aligned(state, 16)));
#define PN_LAUNCH(V, G) rms_seam_kernel<TA, TO, V, G><<<n, PN_THREADS, 0, stream>>>(A)
  JLLM_DISPATCH_1(a_dtype, TA, {
    JLLM_DISPATCH_1(out_dtype, TO, {
      if (wide && d <= PN_THREADS * 4)
        PN_LAUNCH(4, 1);
      else if (wide && d <= PN_THREADS * 8)
        PN_LAUNCH(4, 2);
      else if (wide && d <= PN_THREADS * 16)
        PN_LAUNCH(4, 4);
      else if (wide)
        PN_LAUNCH(4, 8);
      else if (d <= PN_THREADS * 4)
        PN_LAUNCH(1, 4);
      else if (d <= PN_THREADS * 16)
        PN_LAUNCH(1, 16);
      else
        PN_LAUNCH(1, 32);
    })
  })
#undef PN_LAUNCH
  JLLM_CHECK_LAUNCH("rms_seam");
  return 0;
}

// ---------------------------------------------------------------------------------------------------------------------

template <typename TO, int V>
__global__ __launch_bounds__(PN_THREADS) void token_shift_kernel(const float* __restrict__ h, int d, const float* __restrict__ mu,
                                                                 float* state, const int* __restrict__ row_req,
                                                                 const int* __restrict__ state_slots, TO* __restrict__ out,
                                                                 int ldo, int advance) {
  const int t = blockIdx.x;
  const int i = (blockIdx.y * PN_THREADS + threadIdx.x) * V;
  if (i >= d) return;
  const int req = row_req[t];
  const bool first = t == 0 || row_req[t - 1] != req;
  float* st = state + (size_t)state_slots[req] * d;
  float x[V], p[V], m[V], o[V];
  pn_load<V>(h + (size_t)t * d + i, x);
  pn_load<V>((first ? st : h + (size_t)(t - 1) * d) + i, p);
  pn_load<V>(mu + i, m);
#pragma unroll
  for (int e = 0; e < V; ++e) o[e] = x[e] + (p[e] - x[e]) * m[e];
  pn_store<V>(out + (size_t)t * ldo + i, o);
  if (advance) pn_store<V>(st + i, x);  // every request has this one row: nobody else reads its state
}

// the request's last row of the step becomes its state
template <int V>
__global__ __launch_bounds__(PN_THREADS) void token_shift_advance_kernel(const float* __restrict__ h, int n, int d, float* state,
                                                                         const int* __restrict__ row_req,
                                                                         const int* __restrict__ state_slots) {
  const int t = blockIdx.x;
  const int req = row_req[t];
  if (t + 1 < n && row_req[t + 1] == req) return;
  const int i = (blockIdx.y * PN_THREADS + threadIdx.x) * V;
  if (i >= d) return;
  float x[V];
  pn_load<V>(h + (size_t)t * d + i, x);
  pn_store<V>(state + (size_t)state_slots[req] * d + i, x);
}

extern "C" int jllm_token_shift(const float* h, int n, int n_requests, int d, const float* mu, float* state, const int* row_req,
                                const int* state_slots, void* out, int ldo, int out_dtype, hipStream_t stream) {
  if (n <= 0) return 0;
  if (d <= 0 || ldo < d || n_requests <= 0 || n_requests > n) JLLM_FAIL("token_shift: rows of %d into %d, %d requests in %d rows", d, ldo, n_requests, n);
  if (!h || !mu || !state || !row_req || !state_slots || !out) JLLM_FAIL("token_shift: a missing operand");
  const int single = n == n_requests;
  const bool wide = d % 4 == 0 && ldo % 4 == 0 && pn_aligned(h, 16) && pn_aligned(mu, 16) && pn_aligned(state, 16) &&
                    pn_aligned(out, out_dtype == JLLM_F32 ? 16 : 8);
  const int per = PN_THREADS * (wide ? 4 : 1);
  const dim3 grid(n, (d + per - 1) / per);
  JLLM_DISPATCH_1(out_dtype, TO, {
    if (wide)
      token_shift_kernel<TO, 4><<<grid, PN_THREADS, 0, stream>>>(h, d, mu, state, row_req, state_slots, (TO*)out, ldo, single);
    else
      token_shift_kernel<TO, 1><<<grid, PN_THREADS, 0, stream>>>(h, d, mu, state, row_req, state_slots, (TO*)out, ldo, single);
  })
  if (!single) {
    if (wide)
      token_shift_advance_kernel<4><<<grid, PN_THREADS, 0, stream>>>(h, n, d, state, row_req, state_slots);
    else
      token_shift_advance_kernel<1><<<grid, PN_THREADS, 0, stream>>>(h, n, d, state, row_req, state_slots);
  }
  JLLM_CHECK_LAUNCH("token_shift");
  return 0;
}
