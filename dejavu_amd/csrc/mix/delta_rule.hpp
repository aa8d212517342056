// Gated delta rule with one decay per head and key channel; the state is fp32 and stays in registers while a
// portion is walked.
//
//   S <- diag(g) S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q
//
// The columns of S (value channels) are independent: a workgroup owns 16 columns of one head, a row of 16 lanes
// one column, a lane the key channels 64 c + 4 s .. + 3 (s: lane of the row).  Both reductions over the key
// channels are taken of the decayed state, o = (diag(g) S)^T q + (k . q) u, so a token has one dependent reduction.
// State layout [heads][vdim][dim] (key channels contiguous).
#pragma once
#include "elem.hpp"

namespace dv {

// What a lane needs of one token: its E key channels of q, k and the decays, and the scalars of its column.
template <int E>
struct DeltaToken {
  float4_t q[E / 4], k[E / 4], g[E / 4];
  float v, beta, kq;
  __device__ __forceinline__ void load(const float* qp, const float* kp, const float* gp, int sub, float v_, float beta_,
                                       float kq_) {
#pragma unroll
    for (int c = 0; c < E / 4; ++c) {
      k[c] = *reinterpret_cast<const float4_t*>(kp + c * 64 + sub * 4);
      g[c] = *reinterpret_cast<const float4_t*>(gp + c * 64 + sub * 4);
      q[c] = *reinterpret_cast<const float4_t*>(qp + c * 64 + sub * 4);
    }
    v = v_;
    beta = beta_;
    kq = kq_;
  }
};

// One token; S: the E key channels of the lane's column.  Returns the read-out of the column.
template <int E>
__device__ __forceinline__ float delta_step(float (&S)[E], const DeltaToken<E>& t) {
  float dk[4] = {0.f, 0.f, 0.f, 0.f}, dq[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int c = 0; c < E / 4; ++c)
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      S[c * 4 + e] *= t.g[c][e];
      dk[e] = __builtin_fmaf(S[c * 4 + e], t.k[c][e], dk[e]);
      dq[e] = __builtin_fmaf(S[c * 4 + e], t.q[c][e], dq[e]);
    }
  const float sk = row16_sum((dk[0] + dk[1]) + (dk[2] + dk[3]));
  const float sq = row16_sum((dq[0] + dq[1]) + (dq[2] + dq[3]));
  const float u = t.beta * (t.v - sk);
#pragma unroll
  for (int c = 0; c < E / 4; ++c)
#pragma unroll
    for (int e = 0; e < 4; ++e) S[c * 4 + e] = __builtin_fmaf(t.k[c][e], u, S[c * 4 + e]);
  return __builtin_fmaf(t.kq, u, sq);
}

using DeltaArgs = dvDeltaArgs;

template <int E>
__device__ __forceinline__ void load_state(float (&S)[E], const float* __restrict__ p, int sub, int dim_s, bool ok) {
#pragma unroll
  for (int c = 0; c < E / 4; ++c) {
    const int d = c * 64 + sub * 4;
    float4_t t = {0.f, 0.f, 0.f, 0.f};
    if (ok && d < dim_s) t = *reinterpret_cast<const float4_t*>(p + d);
#pragma unroll
    for (int e = 0; e < 4; ++e) S[c * 4 + e] = t[e];
  }
}
template <int E>
__device__ __forceinline__ void store_state(const float (&S)[E], float* __restrict__ p, int sub, int dim_s, bool ok) {
#pragma unroll
  for (int c = 0; c < E / 4; ++c) {
    const int d = c * 64 + sub * 4;
    if (ok && d < dim_s) *reinterpret_cast<float4_t*>(p + d) = float4_t{S[c * 4], S[c * 4 + 1], S[c * 4 + 2], S[c * 4 + 3]};
  }
}

constexpr int kDeltaTokens = 16;  // tokens staged at a time (one 16-lane row each for k . q)
constexpr int kDeltaCols = 16;    // columns of S per workgroup

// A portion of n tokens.  Grid: heads * ceil(vdim_s / 16) workgroups, head fastest.
template <int E>
__global__ __launch_bounds__(256) void delta_scan_kernel(DeltaArgs a) {
  constexpr int D = 16 * E, TC = kDeltaTokens;
  constexpr int V4 = TC * D / 4 / 256;  // float4 per thread and tensor (E / 4)
  constexpr int NB = E <= 8 ? 2 : 1;    // staging buffers
  __shared__ __attribute__((aligned(16))) float sq[NB][TC][D], sk[NB][TC][D], sg[NB][TC][D];
  __shared__ float sv[NB][TC][kDeltaCols], sb[NB][TC], skq[NB][TC];
  const int head = blockIdx.x % a.heads, tile = blockIdx.x / a.heads;
  const int kvh = head / (a.heads / a.kv_heads);
  const int tid = threadIdx.x, sub = tid & 15;
  const int colw = tid >> 4, col = tile * kDeltaCols + colw;  // the 16 rows of 16 lanes: one column each
  const bool col_ok = col < a.vdim_s;
  float S[E];
  float* sp = a.S + ((int64_t)head * a.vdim_s + (col_ok ? col : 0)) * a.dim_s;
  load_state<E>(S, sp, sub, a.dim_s, col_ok);

  float4_t rq[V4], rk[V4], rg[V4];
  float rv, rb = 0.f;
  auto fetch = [&](int t0) {
#pragma unroll
    for (int i = 0; i < V4; ++i) {
      const int at = (i * 256 + tid) * 4, t = at / D, d = at % D;
      const bool ok = t0 + t < a.n && d < a.dim_s;
      const float4_t z = {0.f, 0.f, 0.f, 0.f};
      const int64_t kvat = ((int64_t)(t0 + t) * a.kv_heads + kvh) * a.dim_s + d;
      rq[i] = ok ? *reinterpret_cast<const float4_t*>(a.q + kvat) : z;
      rk[i] = ok ? *reinterpret_cast<const float4_t*>(a.k + kvat) : z;
      rg[i] = ok ? *reinterpret_cast<const float4_t*>(a.g + ((int64_t)(t0 + t) * a.heads + head) * a.dim_s + d) : z;
    }
    const int t = t0 + (tid >> 4), c = tile * kDeltaCols + sub;
    rv = (t < a.n && c < a.vdim_s) ? a.v[((int64_t)t * a.heads + head) * a.vdim_s + c] : 0.f;
    if (sub == 0) rb = t < a.n ? a.beta[(int64_t)t * a.heads + head] : 0.f;
  };
  auto put = [&](int buf) {
#pragma unroll
    for (int i = 0; i < V4; ++i) {
      const int at = (i * 256 + tid) * 4;
      *reinterpret_cast<float4_t*>(&sq[buf][0][0] + at) = rq[i];
      *reinterpret_cast<float4_t*>(&sk[buf][0][0] + at) = rk[i];
      *reinterpret_cast<float4_t*>(&sg[buf][0][0] + at) = rg[i];
    }
    sv[buf][tid >> 4][sub] = rv;
    if (sub == 0) sb[buf][tid >> 4] = rb;
  };
  auto dot_kq = [&](int buf) {
    float d = 0.f;
    const int t = tid >> 4;
#pragma unroll
    for (int c = 0; c < E / 4; ++c) {
      const float4_t x = *reinterpret_cast<const float4_t*>(&sk[buf][t][c * 64 + sub * 4]);
      const float4_t y = *reinterpret_cast<const float4_t*>(&sq[buf][t][c * 64 + sub * 4]);
#pragma unroll
      for (int e = 0; e < 4; ++e) d = __builtin_fmaf(x[e], y[e], d);
    }
    d = row16_sum(d);
    if (sub == 0) skq[buf][t] = d;
  };

  fetch(0);
  put(0);
  __syncthreads();
  dot_kq(0);
  __syncthreads();
  for (int t0 = 0, buf = 0; t0 < a.n; t0 += TC, buf = (buf + 1) % NB) {
    const bool more = t0 + TC < a.n;
    if (more) fetch(t0 + TC);
    const int cnt = a.n - t0 < TC ? a.n - t0 : TC;
    float mine = 0.f;  // lane s keeps the read-out of token s
    DeltaToken<E> cur, nxt;
    auto get = [&](DeltaToken<E>& d, int t) {
      d.load(sq[buf][t], sk[buf][t], sg[buf][t], sub, sv[buf][t][colw], sb[buf][t], skq[buf][t]);
    };
    auto run = [&](const DeltaToken<E>& d, int t) {
      const float o = delta_step<E>(S, d);
      if (sub == t) mine = o;
    };
    get(cur, 0);
    if (cnt == TC) {  // the operands of a token are requested one token ahead
#pragma unroll
      for (int t = 0; t < TC; t += 2) {
        get(nxt, t + 1);
        __builtin_amdgcn_sched_barrier(0);
        run(cur, t);
        __builtin_amdgcn_sched_barrier(0);
        if (t + 2 < TC) get(cur, t + 2);
        __builtin_amdgcn_sched_barrier(0);
        run(nxt, t + 1);
        __builtin_amdgcn_sched_barrier(0);
      }
    } else {
      for (int t = 0; t < cnt; ++t) {
        get(cur, t);
        run(cur, t);
      }
    }
    if (col_ok && sub < cnt) a.o[((int64_t)(t0 + sub) * a.heads + head) * a.vdim_s + col] = mine;
    if (more) {
      const int nb = (buf + 1) % NB;
      if (NB == 1) __syncthreads();  // everybody is done with the only buffer
      put(nb);
      __syncthreads();
      dot_kq(nb);
      __syncthreads();
    }
  }
  store_state<E>(S, sp, sub, a.dim_s, col_ok);
}

// g = exp(-exp(A_log) softplus(z + dt_bias)), beta = sigmoid(b).  Four channels of a head per thread (dim_s % 4 == 0).
template <typename T>
__global__ __launch_bounds__(256) void delta_gates_kernel(const T* __restrict__ z, int64_t ldz, const T* __restrict__ b,
                                                          int64_t ldb, const float* __restrict__ A_log,
                                                          const float* __restrict__ dt_bias, int64_t n, int heads,
                                                          int dim_s, float* __restrict__ g, float* __restrict__ beta) {
  typedef T quad_t __attribute__((ext_vector_type(4)));
  const int per = heads * dim_s / 4;
  const int64_t at = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (at >= n * per) return;
  const int64_t t = at / per;
  const int c = (int)(at % per) * 4, h = c / dim_s;
  const float ea = -exp_f(A_log[h]);
  const quad_t zv = *reinterpret_cast<const quad_t*>(z + t * ldz + c);
  const float4_t bias = *reinterpret_cast<const float4_t*>(dt_bias + c);
  float4_t out;
#pragma unroll
  for (int e = 0; e < 4; ++e) out[e] = exp_f(ea * softplus_f(to_f(zv[e]) + bias[e]));
  *reinterpret_cast<float4_t*>(g + t * heads * dim_s + c) = out;
  if (c % dim_s == 0) beta[t * heads + h] = sigmoid_f(to_f(b[t * ldb + h]));
}

// One decode token straight from the projections (fp32 row `p`: q, k, v after convolution and silu, then the
// logits of beta, then the latent rows of the decay and of the output gate).  A workgroup owns 16 columns of a head
// and also writes their output gates, sigmoid(W_g2 c), for the product that follows.
using DeltaStepArgs = dvDeltaStepArgs;

template <typename T>
__device__ __forceinline__ float dot_row(const T* __restrict__ w, const float* x, int n) {
  float acc = 0.f;
  for (int i = 0; i < n; i += 8) {
    Pack8<T> v;
    v.load(w + i);
#pragma unroll
    for (int e = 0; e < 8; ++e) acc = __builtin_fmaf(v.get(e), x[i + e], acc);
  }
  return acc;
}

template <typename T, int E>
__global__ __launch_bounds__(256) void delta_decode_kernel(DeltaStepArgs a) {
  constexpr int D = 16 * E;
  extern __shared__ __attribute__((aligned(16))) unsigned char smem_raw[];
  float* lat = reinterpret_cast<float*>(smem_raw);  // rank_a + rank_g latents, as the products see them
  __shared__ __attribute__((aligned(16))) float sq[D], sk[D], sg[D];
  __shared__ float skq;
  const int head = blockIdx.x % a.heads, tile = blockIdx.x / a.heads;
  const int kvh = head / (a.heads / a.kv_heads);
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, sub = tid & 15;
  const int col = tile * kDeltaCols + (tid >> 4);
  const bool col_ok = col < a.vdim_s;
  float S[E];
  float* sp = a.S + ((int64_t)head * a.vdim_s + (col_ok ? col : 0)) * a.dim_s;
  load_state<E>(S, sp, sub, a.dim_s, col_ok);  // requested before the small products below
  for (int i = tid; i < a.rank_a; i += 256) lat[i] = to_f(from_f<T>(a.p[a.off_a + i]));
  for (int i = tid; i < a.rank_g; i += 256) lat[a.rank_a + i] = to_f(from_f<T>(a.p[a.off_g + i]));
  if (wave < 2) {
    const float* src = a.p + (wave ? a.off_k : 0) + (int64_t)kvh * a.dim_s;
    float* dst = wave ? sk : sq;
    float x[(D + 63) / 64], ss = 0.f;
#pragma unroll
    for (int i = 0; i < (D + 63) / 64; ++i) {
      const int d = lane + i * 64;
      x[i] = d < a.dim_s ? src[d] : 0.f;
      ss = __builtin_fmaf(x[i], x[i], ss);
    }
    float s = 1.f / sqrtf(wave_sum(ss) + 1e-6f);
    if (!wave) s *= 1.f / sqrtf((float)a.dim);
#pragma unroll
    for (int i = 0; i < (D + 63) / 64; ++i)
      if (lane + i * 64 < D) dst[lane + i * 64] = x[i] * s;
  }
  __syncthreads();
  // decays: two lanes per key channel
  const T* Wa = reinterpret_cast<const T*>(a.Wa);
  const T* Wg = reinterpret_cast<const T*>(a.Wg);
  const float ea = exp_f(a.A_log[head]);
  const int half = tid & 1, cut = (a.rank_a / 2 + 7) / 8 * 8;
  for (int d = tid >> 1; d < D; d += 128) {
    float z = 0.f;
    if (d < a.dim_s) {
      const T* w = Wa + (int64_t)(head * a.dim_s + d) * a.rank_a;
      z = half ? dot_row<T>(w + cut, lat + cut, a.rank_a - cut) : dot_row<T>(w, lat, cut);
    }
    z = dpp_add<0xB1>(z);
    if (half == 0) sg[d] = d < a.dim_s ? exp_f(-ea * softplus_f(z + a.dt_bias[head * a.dim_s + d])) : 0.f;
  }
  // output gates: a row of 16 lanes per column
  float gz = 0.f;
  if (col_ok) {
    const T* w = Wg + (int64_t)(head * a.vdim_s + col) * a.rank_g;
    for (int i = sub * 8; i < a.rank_g; i += 128) {
      Pack8<T> v;
      v.load(w + i);
#pragma unroll
      for (int e = 0; e < 8; ++e) gz = __builtin_fmaf(v.get(e), lat[a.rank_a + i + e], gz);
    }
  }
  gz = row16_sum(gz);
  if (wave == 0) {
    float d = 0.f;
    for (int i = lane; i < D; i += 64) d = __builtin_fmaf(sq[i], sk[i], d);
    d = wave_sum(d);
    if (lane == 0) skq = d;
  }
  __syncthreads();
  const float v = col_ok ? a.p[a.off_v + (int64_t)head * a.vdim_s + col] : 0.f;
  const float beta = sigmoid_f(a.p[a.off_b + head]);
  DeltaToken<E> tok;
  tok.load(sq, sk, sg, sub, v, beta, skq);
  const float o = delta_step<E>(S, tok);
  store_state<E>(S, sp, sub, a.dim_s, col_ok);
  if (col_ok && sub == 0) {
    a.o[(int64_t)head * a.vdim_s + col] = o;
    a.gate[(int64_t)head * a.vdim_s + col] = sigmoid_f(gz);
  }
}

}  // namespace dv
