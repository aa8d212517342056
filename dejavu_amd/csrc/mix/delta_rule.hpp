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
// T and M depend on no state: one kernel makes them for all chunks at once.  The second kernel carries the state from
// chunk to chunk; its products run on the fp32 matrix instructions.  A decode step uses the recurrence itself.
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

// T and M of a chunk and head: tm[(chunk * heads + head) * 512] = T [16][16], then M [16][16].  A row of 16 lanes owns
// key j and walks the later tokens.  Grid: (heads, chunks); D = 16 E >= dim_s.
template <int E>
__global__ __launch_bounds__(256) void delta_chunk_kernel(DeltaArgs a) {
  constexpr int D = 16 * E, C = kDeltaChunk;
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
    *reinterpret_cast<float4_t*>(sg + at) = ok ? g : z;
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
  float* out = a.tm + ((int64_t)blockIdx.y * a.heads + head) * 512;
  if (tid < C) {  // column tid of T by forward substitution
    float x[C];
#pragma unroll
    for (int i = 0; i < C; ++i) {
      float v = i == tid ? sb[i] : 0.f;
#pragma unroll
      for (int k = 0; k < i; ++k) v = __builtin_fmaf(-L[i][k], x[k], v);
      x[i] = v;
      out[i * C + tid] = v;
    }
  }
  out[256 + tid] = M[j][sub];
}

// Chunk after chunk for 16 columns of a head.  Wave w owns key channels [16 NT w, 16 NT (w + 1)) of the state, as
// accumulators of the 16x16x4 products: element i of a lane is channel 4 (lane / 16) + i of a tile, column lane % 16,
// which is also the operand layout of the products with Kt and Qt when their channels are taken in that order.  The
// four waves' partial products meet in LDS once per chunk; U is then made by every wave for itself.
template <int NT>
struct DeltaChunkLds {
  static constexpr int D = 64 * NT, KL = D + 4, TL = 20;
  float kt[16 * KL], qt[16 * KL];  // [token][channel]
  float kh[D * TL];                // [channel][token]
  float tmat[16 * TL], mmat[16 * TL];
  float v[16 * 16];                // [token][column]
  float gc[D];                     // decay over the whole chunk
};
template <int NT>
constexpr size_t delta_scan_lds_bytes() {
  return 2 * sizeof(DeltaChunkLds<NT>) + 2 * 4 * 2 * 64 * 16;  // two stages; partial products, two stages
}

// Grid: heads * ceil(vdim_s / 16), head fastest (the workgroups of a head share an XCD's L2 when heads % 8 == 0).
template <int NT>
__global__ __launch_bounds__(256) void delta_scan_kernel(DeltaArgs a) {
  using Lds = DeltaChunkLds<NT>;
  constexpr int D = Lds::D, KL = Lds::KL, TL = Lds::TL, C = kDeltaChunk;
  constexpr int IT = (2 * D + 255) / 256;  // (role, channel) items per thread
  extern __shared__ __attribute__((aligned(16))) unsigned char smem_raw[];
  Lds* st = reinterpret_cast<Lds*>(smem_raw);
  float4_t* part = reinterpret_cast<float4_t*>(smem_raw + 2 * sizeof(Lds));  // [stage][wave][2][64]
  const int head = blockIdx.x % a.heads, tile = blockIdx.x / a.heads;
  const int kvh = head / (a.heads / a.kv_heads);
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int l16 = lane & 15, q4 = lane >> 4;
  const int col = tile * kDeltaCols + l16;
  const bool col_ok = col < a.vdim_s;
  float* sp = a.S + ((int64_t)head * a.vdim_s + (col_ok ? col : 0)) * a.dim_s;
  float4_t S[NT];
#pragma unroll
  for (int t = 0; t < NT; ++t) {
    const int d = (wave * NT + t) * 16 + q4 * 4;
    S[t] = (col_ok && d < a.dim_s) ? *reinterpret_cast<const float4_t*>(sp + d) : float4_t{0.f, 0.f, 0.f, 0.f};
  }

  // staging: role 0 makes Kt and Qt of a channel, role 1 Kh and the chunk's decay
  float rg[IT][C], rk[IT][C], rq[IT][C], rtm[2], rv;
  const int gs = a.heads * a.dim_s, ks_ = a.kv_heads * a.dim_s;  // elements between tokens
  const int vc = min(tile * kDeltaCols + (tid & 15), a.vdim_s - 1);
  auto fetch = [&](int t0) {
    const float* gp = a.g + (int64_t)t0 * gs + head * a.dim_s;
    const float* kp = a.k + (int64_t)t0 * ks_ + kvh * a.dim_s;
    const float* qp = a.q + (int64_t)t0 * ks_ + kvh * a.dim_s;
    const int last = a.n - 1 - t0;
#pragma unroll
    for (int it = 0; it < IT; ++it) {
      const int d = min((it * 256 + tid) % D, a.dim_s - 1);
#pragma unroll
      for (int t = 0; t < C; ++t) {
        const int row = min(t, last);
        rg[it][t] = gp[row * gs + d];
        rk[it][t] = kp[row * ks_ + d];
        rq[it][t] = qp[row * ks_ + d];
      }
    }
    const float* tm = a.tm + ((int64_t)(t0 / C) * a.heads + head) * 512;
    rtm[0] = tm[tid];
    rtm[1] = tm[256 + tid];
    rv = a.v[((int64_t)t0 + min(tid >> 4, last)) * a.heads * a.vdim_s + head * a.vdim_s + vc];
  };
  auto put = [&](Lds& b, int t0) {
    // what was read past the end of the portion or of the channels
    const int cnt = a.n - t0;
#pragma unroll
    for (int it = 0; it < IT; ++it) {
      const bool in = (it * 256 + tid) % D < a.dim_s;
#pragma unroll
      for (int t = 0; t < C; ++t) {
        if (!in || t >= cnt) {
          rg[it][t] = 1.f;
          rk[it][t] = 0.f;
          rq[it][t] = 0.f;
        }
      }
    }
    if ((tid >> 4) >= cnt) rv = 0.f;
#pragma unroll
    for (int it = 0; it < IT; ++it) {
      const int item = it * 256 + tid, role = item / D, d = item % D;
      if (item < 2 * D) {
        if (role == 0) {
          float p = 1.f;
#pragma unroll
          for (int t = 0; t < C; ++t) {
            p *= rg[it][t];
            b.kt[t * KL + d] = p * rk[it][t];
            b.qt[t * KL + d] = p * rq[it][t];
          }
        } else {
          float p = 1.f;
          float kh[C];
#pragma unroll
          for (int t = C - 1; t >= 0; --t) {
            kh[t] = p * rk[it][t];
            p *= rg[it][t];
          }
          b.gc[d] = p;
#pragma unroll
          for (int t = 0; t < C; t += 4)
            *reinterpret_cast<float4_t*>(&b.kh[d * TL + t]) = float4_t{kh[t], kh[t + 1], kh[t + 2], kh[t + 3]};
        }
      }
    }
    b.tmat[(tid >> 4) * TL + (tid & 15)] = rtm[0];
    b.mmat[(tid >> 4) * TL + (tid & 15)] = rtm[1];
    b.v[tid] = rv;
  };

  fetch(0);
  put(st[0], 0);
  __syncthreads();
  for (int t0 = 0, buf = 0; t0 < a.n; t0 += C, buf ^= 1) {
    const Lds& b = st[buf];
    const bool more = t0 + C < a.n;
    if (more) fetch(t0 + C);
    // partial Kt S and Qt S over this wave's channels
    float4_t ks = {0.f, 0.f, 0.f, 0.f}, qs = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int t = 0; t < NT; ++t) {
      const int d = (wave * NT + t) * 16 + q4 * 4;
      const float4_t kt = *reinterpret_cast<const float4_t*>(&b.kt[l16 * KL + d]);
      const float4_t qt = *reinterpret_cast<const float4_t*>(&b.qt[l16 * KL + d]);
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        ks = __builtin_amdgcn_mfma_f32_16x16x4f32(kt[i], S[t][i], ks, 0, 0, 0);
        qs = __builtin_amdgcn_mfma_f32_16x16x4f32(qt[i], S[t][i], qs, 0, 0, 0);
      }
    }
    float4_t* pp = part + buf * 512;
    pp[wave * 128 + lane] = ks;
    pp[wave * 128 + 64 + lane] = qs;
    __syncthreads();
    float4_t w;  // V - Kt S: tokens 4 q4 .. + 3 of this lane's column
    const float4_t sum = (pp[lane] + pp[128 + lane]) + (pp[256 + lane] + pp[384 + lane]);
#pragma unroll
    for (int i = 0; i < 4; ++i) w[i] = b.v[(q4 * 4 + i) * 16 + l16] - sum[i];
    const float4_t tm = *reinterpret_cast<const float4_t*>(&b.tmat[l16 * TL + q4 * 4]);
    float4_t u = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int i = 0; i < 4; ++i) u = __builtin_amdgcn_mfma_f32_16x16x4f32(tm[i], w[i], u, 0, 0, 0);
    if (wave == 3) {
      float4_t o = (pp[64 + lane] + pp[192 + lane]) + (pp[320 + lane] + pp[448 + lane]);
      const float4_t mm = *reinterpret_cast<const float4_t*>(&b.mmat[l16 * TL + q4 * 4]);
#pragma unroll
      for (int i = 0; i < 4; ++i) o = __builtin_amdgcn_mfma_f32_16x16x4f32(mm[i], u[i], o, 0, 0, 0);
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int t = t0 + q4 * 4 + i;
        if (col_ok && t < a.n) a.o[((int64_t)t * a.heads + head) * a.vdim_s + col] = o[i];
      }
    }
#pragma unroll
    for (int t = 0; t < NT; ++t) {
      const int d0 = (wave * NT + t) * 16;
      const float4_t gc = *reinterpret_cast<const float4_t*>(&b.gc[d0 + q4 * 4]);
      const float4_t kh = *reinterpret_cast<const float4_t*>(&b.kh[(d0 + l16) * TL + q4 * 4]);
      S[t] *= gc;
#pragma unroll
      for (int i = 0; i < 4; ++i) S[t] = __builtin_amdgcn_mfma_f32_16x16x4f32(kh[i], u[i], S[t], 0, 0, 0);
    }
    if (more) put(st[buf ^ 1], t0 + C);  // that stage was read before the barrier above
    __syncthreads();
  }
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
