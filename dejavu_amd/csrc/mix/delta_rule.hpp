// Gated delta rule with one decay per head and key channel, in fp32.
//
//   S <- diag(g) S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q
//
// A portion is walked in chunks of 16 tokens.  With P(i, j) = g_{j+1} .. g_i per channel (products, never exponentials
// of summed logarithms: they are as exact as the token-by-token recurrence and cannot overflow) and S_0 the state at
// the start of the chunk,
//
//   L[i, j] = sum_d k_i k_j P(i, j)  (j < i)     M[i, j] = sum_d q_i k_j P(i, j)  (j <= i)
//   U = T (V - Kt S_0),  T = (1 + diag(beta) L)^-1 diag(beta),  Kt_i = P(i, 0) k_i  (g_1 included)
//   O = Qt S_0 + M U,    S = P(16, 0) S_0 + Kh^T U,             Kh_j = P(16, j) k_j
//
// Everything but U, O and S depends on no state: one kernel makes it for many chunks at once.  The second kernel
// carries the state from chunk to chunk; its products run on the fp32 matrix instructions.  A decode step uses the
// recurrence itself.
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

constexpr int kDeltaCols = 16;   // columns of S per workgroup
constexpr int kDeltaChunk = 16;  // tokens per chunk

// What the first kernel leaves for a chunk and head, in floats and in the order the second kernel's lanes load it
// (lane = 16 q + r, four floats per lane, 256 floats per operand): for every tile of 16 channels Kt and Qt (token r,
// channels 4 q ..), Kh (channel r, tokens 4 q ..); then T and M (row r, columns 4 q ..); then the decay over the chunk
// per channel.  D = 64 NT >= dim_s.
template <int NT>
struct DeltaChunk {
  static constexpr int D = 64 * NT;
  static constexpr int kt = 0, qt = 16 * D, kh = 32 * D, t = 48 * D, m = t + 256, gc = m + 256, floats = gc + D;
};

// A row of 16 lanes owns key j and walks the later tokens for T and M; then a thread owns a channel for the rest.
// Grid: (heads, chunks).
template <int NT>
__global__ __launch_bounds__(256) void delta_chunk_kernel(DeltaArgs a) {
  using Out = DeltaChunk<NT>;
  constexpr int E = 4 * NT, D = 64 * NT, C = kDeltaChunk;
  extern __shared__ __attribute__((aligned(16))) unsigned char smem_raw[];
  float* sq = reinterpret_cast<float*>(smem_raw);  // [16][D] each
  float* sk = sq + C * D;
  float* sg = sk + C * D;
  __shared__ __attribute__((aligned(16))) float L[C][C], M[C][C];
  __shared__ float sb[C];
  const int head = blockIdx.x, t0 = blockIdx.y * C, kvh = head / (a.heads / a.kv_heads);
  const int tid = threadIdx.x, sub = tid & 15, j = tid >> 4;
#pragma unroll
  for (int i = 0; i < E / 4; ++i) {
    const int at = (i * 256 + tid) * 4, t = at / D, d = at % D;
    const bool ok = t0 + t < a.n && d < a.dim_s;
    const int64_t row = min(t0 + t, a.n - 1);
    const int dc = min(d, a.dim_s - 4);
    const float4_t z = {0.f, 0.f, 0.f, 0.f};
    const float4_t q = *reinterpret_cast<const float4_t*>(a.q + (row * a.kv_heads + kvh) * a.dim_s + dc);
    const float4_t k = *reinterpret_cast<const float4_t*>(a.k + (row * a.kv_heads + kvh) * a.dim_s + dc);
    const float4_t g = *reinterpret_cast<const float4_t*>(a.g + (row * a.heads + head) * a.dim_s + dc);
    *reinterpret_cast<float4_t*>(sq + at) = ok ? q : z;
    *reinterpret_cast<float4_t*>(sk + at) = ok ? k : z;
    *reinterpret_cast<float4_t*>(sg + at) = ok ? g : float4_t{1.f, 1.f, 1.f, 1.f};  // past the end: nothing decays
  }
  if (tid < C) sb[tid] = t0 + tid < a.n ? a.beta[(int64_t)(t0 + tid) * a.heads + head] : 0.f;
  L[j][sub] = 0.f;
  M[j][sub] = 0.f;
  __syncthreads();
  float4_t p[E / 4];  // k_j P(i, j)
#pragma unroll
  for (int c = 0; c < E / 4; ++c) p[c] = *reinterpret_cast<const float4_t*>(sk + j * D + c * 64 + sub * 4);
  for (int i = j; i < C; ++i) {
    float kk = 0.f, qk = 0.f;
#pragma unroll
    for (int c = 0; c < E / 4; ++c) {
      const int at = i * D + c * 64 + sub * 4;
      const float4_t qv = *reinterpret_cast<const float4_t*>(sq + at), kv = *reinterpret_cast<const float4_t*>(sk + at);
      if (i > j) p[c] *= *reinterpret_cast<const float4_t*>(sg + at);
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        kk = __builtin_fmaf(p[c][e], kv[e], kk);
        qk = __builtin_fmaf(p[c][e], qv[e], qk);
      }
    }
    kk = row16_sum(kk);
    qk = row16_sum(qk);
    if (sub == 0) {
      M[i][j] = qk;
      if (i > j) L[i][j] = sb[i] * kk;
    }
  }
  __syncthreads();
  float* out = a.tm + ((int64_t)blockIdx.y * a.heads + head) * Out::floats;
  if (tid < C) {  // column tid of T by forward substitution
    float x[C];
#pragma unroll
    for (int i = 0; i < C; ++i) {
      float v = i == tid ? sb[i] : 0.f;
#pragma unroll
      for (int k = 0; k < i; ++k) v = __builtin_fmaf(-L[i][k], x[k], v);
      x[i] = v;
      out[Out::t + ((tid >> 2) * 16 + i) * 4 + (tid & 3)] = v;
    }
  }
  out[Out::m + ((sub >> 2) * 16 + j) * 4 + (sub & 3)] = M[j][sub];
  // a thread per channel makes Kt and Qt, another one Kh; they change places with k, q and g in LDS
  constexpr int IT = (2 * D + 255) / 256;
  float r0[IT][C], r1[IT][C];
#pragma unroll
  for (int it = 0; it < IT; ++it) {
    const int item = it * 256 + 255 - tid, d = item % D;  // the first wave, busy with T, comes last
    float p = 1.f;
    if (item < D) {
#pragma unroll
      for (int t = 0; t < C; ++t) {
        p *= sg[t * D + d];
        r0[it][t] = p * sk[t * D + d];
        r1[it][t] = p * sq[t * D + d];
      }
    } else if (item < 2 * D) {
#pragma unroll
      for (int t = C - 1; t >= 0; --t) {
        r0[it][t] = p * sk[t * D + d];
        p *= sg[t * D + d];
      }
      out[Out::gc + d] = p;
    }
  }
  __syncthreads();
#pragma unroll
  for (int it = 0; it < IT; ++it) {
    const int item = it * 256 + 255 - tid, d = item % D;
#pragma unroll
    for (int t = 0; t < C; ++t) {
      if (item < D) {
        sk[t * D + d] = r0[it][t];
        sq[t * D + d] = r1[it][t];
      } else if (item < 2 * D) {
        sg[t * D + d] = r0[it][t];
      }
    }
  }
  __syncthreads();
  for (int i = tid; i < 4 * D; i += 256) {
    const int tile = i >> 6, q = (i >> 4) & 3, r = i & 15;
    *reinterpret_cast<float4_t*>(out + Out::kt + i * 4) = *reinterpret_cast<const float4_t*>(sk + r * D + tile * 16 + q * 4);
    *reinterpret_cast<float4_t*>(out + Out::qt + i * 4) = *reinterpret_cast<const float4_t*>(sq + r * D + tile * 16 + q * 4);
    const float* g = sg + q * 4 * D + tile * 16 + r;
    *reinterpret_cast<float4_t*>(out + Out::kh + i * 4) = float4_t{g[0], g[D], g[2 * D], g[3 * D]};
  }
}

// Chunk after chunk for 16 columns of a head.  Wave w owns key channels [16 NT w, 16 NT (w + 1)) of the state, as
// accumulators of the 16x16x4 products: element i of a lane is channel 4 (lane / 16) + i of a tile, column lane % 16,
// which is also the operand layout of the products with Kt and Qt when their channels are taken in that order.  All
// operands are loaded by the lanes that use them, a chunk ahead.  The waves' parts of Kt S meet in LDS once per chunk
// and every wave makes U for itself.  A wave's part of O is Qt S over its channels plus every fourth token's share of
// M U; the parts meet at the next chunk's barrier.
template <int NT>
struct DeltaOperands {
  float4_t kt[NT], qt[NT], kh[NT], gc[NT], t;
  float m, v[4];
};

// Grid: heads * ceil(vdim_s / 16), head fastest (the workgroups of a head share an XCD's L2 when heads % 8 == 0).
template <int NT>
__global__ __launch_bounds__(256) void delta_scan_kernel(DeltaArgs a) {
  using In = DeltaChunk<NT>;
  constexpr int C = kDeltaChunk;
  __shared__ __attribute__((aligned(16))) float4_t kpart[2][4][64], opart[2][4][64];
  const int head = blockIdx.x % a.heads, tile = blockIdx.x / a.heads;
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int l16 = lane & 15, q4 = lane >> 4;
  const int col = tile * kDeltaCols + l16;
  const bool col_ok = col < a.vdim_s;
  const int vstep = a.heads * a.vdim_s;
  float* sp = a.S + ((int64_t)head * a.vdim_s + (col_ok ? col : 0)) * a.dim_s;
  float4_t S[NT];
#pragma unroll
  for (int t = 0; t < NT; ++t) {
    const int d = (wave * NT + t) * 16 + q4 * 4;
    S[t] = (col_ok && d < a.dim_s) ? *reinterpret_cast<const float4_t*>(sp + d) : float4_t{0.f, 0.f, 0.f, 0.f};
  }
  const float* vcol = a.v + head * a.vdim_s + min(col, a.vdim_s - 1);
  const int chunks = (a.n + C - 1) / C;
  // rows of V past the end meet zeros of T
  auto load = [&](DeltaOperands<NT>& x, int c) {
    const float* src = a.tm + ((int64_t)c * a.heads + head) * In::floats;
#pragma unroll
    for (int t = 0; t < NT; ++t) {
      const int tt = wave * NT + t;
      x.kt[t] = *reinterpret_cast<const float4_t*>(src + In::kt + tt * 256 + lane * 4);
      x.qt[t] = *reinterpret_cast<const float4_t*>(src + In::qt + tt * 256 + lane * 4);
      x.kh[t] = *reinterpret_cast<const float4_t*>(src + In::kh + tt * 256 + lane * 4);
      x.gc[t] = *reinterpret_cast<const float4_t*>(src + In::gc + tt * 16 + q4 * 4);
    }
    x.t = *reinterpret_cast<const float4_t*>(src + In::t + lane * 4);
    x.m = src[In::m + lane * 4 + wave];
#pragma unroll
    for (int i = 0; i < 4; ++i) x.v[i] = vcol[(int64_t)min(c * C + q4 * 4 + i, a.n - 1) * vstep];
  };
  // read-outs of a chunk: a lane stores token 4 wave + q4 of its column
  const float* op = reinterpret_cast<const float*>(opart) + (wave * 16 + l16) * 4 + q4;
  float* ocol = a.o + (int64_t)head * a.vdim_s + col;
  auto store_o = [&](int c, int par) {
    const float* p = op + par * 1024;
    const int t = c * C + wave * 4 + q4;
    const float o = (p[0] + p[256]) + (p[512] + p[768]);
    if (col_ok && t < a.n) ocol[(int64_t)t * vstep] = o;
  };
  auto step = [&](const DeltaOperands<NT>& x, int c, int par) {
    float4_t ks[NT];
#pragma unroll
    for (int t = 0; t < NT; ++t) ks[t] = float4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
      for (int t = 0; t < NT; ++t) ks[t] = __builtin_amdgcn_mfma_f32_16x16x4f32(x.kt[t][i], S[t][i], ks[t], 0, 0, 0);
#pragma unroll
    for (int t = 1; t < NT; ++t) ks[0] += ks[t];
    kpart[par][wave][lane] = ks[0];
    float4_t qs = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
      for (int t = 0; t < NT; ++t) qs = __builtin_amdgcn_mfma_f32_16x16x4f32(x.qt[t][i], S[t][i], qs, 0, 0, 0);
    __syncthreads();
    const float4_t sum = (kpart[par][0][lane] + kpart[par][1][lane]) + (kpart[par][2][lane] + kpart[par][3][lane]);
    float4_t u = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int i = 0; i < 4; ++i) u = __builtin_amdgcn_mfma_f32_16x16x4f32(x.t[i], x.v[i] - sum[i], u, 0, 0, 0);
#pragma unroll
    for (int t = 0; t < NT; ++t) S[t] *= x.gc[t];
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
      for (int t = 0; t < NT; ++t) S[t] = __builtin_amdgcn_mfma_f32_16x16x4f32(x.kh[t][i], u[i], S[t], 0, 0, 0);
    const float uw = wave == 0 ? u[0] : (wave == 1 ? u[1] : (wave == 2 ? u[2] : u[3]));
    qs = __builtin_amdgcn_mfma_f32_16x16x4f32(x.m, uw, qs, 0, 0, 0);
    if (c > 0) store_o(c - 1, par ^ 1);
    opart[par][wave][lane] = qs;
  };
  DeltaOperands<NT> even, odd;
  load(even, 0);
  for (int c = 0; c < chunks; c += 2) {
    load(odd, min(c + 1, chunks - 1));
    step(even, c, 0);
    if (c + 1 < chunks) {
      load(even, min(c + 2, chunks - 1));
      step(odd, c + 1, 1);
    }
  }
  __syncthreads();
  store_o(chunks - 1, (chunks - 1) & 1);
#pragma unroll
  for (int t = 0; t < NT; ++t) {
    const int d = (wave * NT + t) * 16 + q4 * 4;
    if (col_ok && d < a.dim_s) *reinterpret_cast<float4_t*>(sp + d) = S[t];
  }
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
  for (int i = 0; i < n; i += 64) {  // eight packets requested together
    Pack8<T> v[8];
#pragma unroll
    for (int u = 0; u < 8; ++u) v[u].load(w + min(i + u * 8, n - 8));
#pragma unroll
    for (int u = 0; u < 8; ++u)
      if (i + u * 8 < n) {
#pragma unroll
        for (int e = 0; e < 8; ++e) acc = __builtin_fmaf(v[u].get(e), x[i + u * 8 + e], acc);
      }
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
