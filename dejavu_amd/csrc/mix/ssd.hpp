// Mamba-2 recurrence (one decay per head and token) in fp32.
//
//   S <- a S + dt B x^T;  y = S^T C + D x,  a = exp(-exp(A_log) dt)
//
// A portion is walked in chunks of 64 tokens.  With P(i, j) = a_{j+1} .. a_i (products of the decays, as exact as the
// token-by-token recurrence) and S_0 the state at the start of the chunk,
//
//   Y = diag(P(i, 0)) C S_0 + M X,   M[i, j] = (C_i . B_j) P(i, j) dt_j  (j <= i; D joins the diagonal)
//   S = P(64, 0) S_0 + B^T diag(P(64, j) dt_j) X                          (P(i, 0), P(64, 0): a_1 included)
//
// M and the factors depend on no state: one kernel makes them for all chunks at once, C B^T once for the heads of a
// group that a workgroup takes.  The second kernel carries the state from chunk to chunk.  All products run on the
// fp32 matrix instructions.  A decode step uses the recurrence itself.
// State layout [heads][vdim][state_s].
#pragma once
#include "elem.hpp"

namespace dv {

using SsdArgs = dvSsdArgs;

constexpr int kSsdChunk = 64, kSsdCols = 16;

// What the first kernel leaves for a chunk and head, in floats: the 10 tiles of M on and below the diagonal (row tile r,
// column tile c at r (r + 1) / 2 + c), each in the order in which the second kernel's lanes load it (lane = 16 q + i: row
// i, columns 4 q ..); P(i, 0); P(64, j) dt_j.
struct SsdChunk {
  static constexpr int m = 0, p0 = 2560, e = p0 + 64, floats = e + 64;
};

struct SsdGates {
  float dt, a;  // step size and decay
};
__device__ __forceinline__ SsdGates ssd_gates(float logit, float dt_bias, float A_log) {
  SsdGates g;
  g.dt = softplus_f(logit + dt_bias);
  g.a = exp_f(-exp_f(A_log) * g.dt);
  return g;
}

// Grid: (groups * slices of hp heads, chunks).  Wave w takes row tile (w + chunk) % 4 of M, so that no SIMD gets the
// longest row every time.
template <typename T>
__global__ __launch_bounds__(256) void ssd_chunk_kernel(SsdArgs a, int hp) {
  __shared__ __attribute__((aligned(16))) float tab[4][16][68];  // P(i, j) dt_j of a row tile
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int l16 = lane & 15, q4 = lane >> 4;
  const int rep = a.heads / a.groups, slices = (rep + hp - 1) / hp;
  const int group = blockIdx.x / slices, h0 = group * rep + blockIdx.x % slices * hp;
  const int nh = min(hp, (group + 1) * rep - h0);
  const int t0 = blockIdx.y * kSsdChunk, rt = (wave + blockIdx.y) & 3;
  // logits of the step sizes of the first head, requested before the products
  const T* dtp = reinterpret_cast<const T*>(a.dt) + (int64_t)min(t0 + lane, a.n - 1) * a.lddt;
  float logit = to_f(dtp[h0]);
  const int N = a.state_s;
  const float* Bp[4];
#pragma unroll
  for (int c = 0; c < 4; ++c)
    Bp[c] = a.xbc + (int64_t)min(t0 + c * 16 + l16, a.n - 1) * a.ld + a.off_b + group * N;
  const float* Cp = a.xbc + (int64_t)min(t0 + rt * 16 + l16, a.n - 1) * a.ld + a.off_c + group * N;
  float4_t acc[4];
#pragma unroll
  for (int c = 0; c < 4; ++c) acc[c] = float4_t{0.f, 0.f, 0.f, 0.f};
  for (int k = 0; k < N; k += 16) {
    const int n = min(k + q4 * 4, N - 4);
    float4_t cv = *reinterpret_cast<const float4_t*>(Cp + n), bv[4];
#pragma unroll
    for (int c = 0; c < 4; ++c)
      if (c <= rt) bv[c] = *reinterpret_cast<const float4_t*>(Bp[c] + n);
    if (k + q4 * 4 >= N) cv = float4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int c = 0; c < 4; ++c)
      if (c <= rt) {
#pragma unroll
        for (int i = 0; i < 4; ++i) acc[c] = __builtin_amdgcn_mfma_f32_16x16x4f32(bv[c][i], cv[i], acc[c], 0, 0, 0);
      }
  }
  for (int hi = 0; hi < nh; ++hi) {
    const int h = h0 + hi;
    SsdGates g = ssd_gates(logit, a.dt_bias[h], a.A_log[h]);
    if (hi + 1 < nh) logit = to_f(dtp[h + 1]);
    if (t0 + lane >= a.n) {  // past the end: nothing decays, nothing joins
      g.dt = 0.f;
      g.a = 1.f;
    }
    float* out = a.tm + ((int64_t)blockIdx.y * a.heads + h) * SsdChunk::floats;
    float p = 1.f;  // P(t, lane) once token t has been taken
    auto take = [&](int t) {
      const float at = __int_as_float(__builtin_amdgcn_readlane(__float_as_int(g.a), t));
      p = lane < t ? p * at : p;
    };
#pragma unroll 16
    for (int t = 0; t < rt * 16; ++t) take(t);
#pragma unroll
    for (int r = 0; r < 16; ++r) {
      take(rt * 16 + r);
      tab[wave][r][lane] = lane <= rt * 16 + r ? p * g.dt : 0.f;
    }
    if (rt == 3) {
      out[SsdChunk::e + lane] = p * g.dt;
      float p0 = 1.f;
#pragma unroll 16
      for (int t = 0; t < 64; ++t) {
        const float at = __int_as_float(__builtin_amdgcn_readlane(__float_as_int(g.a), t));
        p0 = lane >= t ? p0 * at : p0;
      }
      out[SsdChunk::p0 + lane] = p0;
    }
    __syncthreads();
#pragma unroll
    for (int c = 0; c < 4; ++c)
      if (c <= rt) {
        float4_t m = acc[c] * *reinterpret_cast<const float4_t*>(&tab[wave][l16][c * 16 + q4 * 4]);
        if (c == rt) {
#pragma unroll
          for (int i = 0; i < 4; ++i)
            if (q4 * 4 + i == l16) m[i] += a.D[h];
        }
        *reinterpret_cast<float4_t*>(out + SsdChunk::m + (rt * (rt + 1) / 2 + c) * 256 + lane * 4) = m;
      }
    __syncthreads();
  }
}

// Chunk after chunk for 16 columns of a head.  Wave w owns channels [16 NT w, 16 NT (w + 1)) of the state as
// accumulators of the 16x16x4 products (element i of a lane: channel 4 (lane / 16) + i of a tile, column lane % 16),
// which is also the operand layout of the product with C when its channels are taken in that order; the waves exchange
// the state through LDS once per chunk, then every wave makes 16 tokens of Y and its own channels of the next state.
// Operands are loaded by the lanes that use them, a chunk ahead: those of the state's own part as soon as it is done with
// them, those of the product with the state after that product.
template <int NT>
struct SsdOperands {
  float4_t c[4 * NT], p0, m[4], e[4];
  float b[NT][4][4], x[4][4], total;
};

// Grid: heads * ceil(vdim / 16), head fastest.
template <int NT>
__global__ __launch_bounds__(256, NT <= 2 ? 2 : 1) void ssd_scan_kernel(SsdArgs a) {
  constexpr int C = kSsdChunk;
  __shared__ __attribute__((aligned(16))) float4_t state[2][4 * NT][64];
  const int head = blockIdx.x % a.heads, tile = blockIdx.x / a.heads;
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int l16 = lane & 15, q4 = lane >> 4, N = a.state_s;
  const int group = head / (a.heads / a.groups);
  const int col = tile * kSsdCols + l16;
  const bool col_ok = col < a.vdim;
  float* sp = a.S + ((int64_t)head * a.vdim + (col_ok ? col : 0)) * N;
  float4_t S[NT];
#pragma unroll
  for (int t = 0; t < NT; ++t) {
    const int n = (wave * NT + t) * 16 + q4 * 4;
    S[t] = (col_ok && n < N) ? *reinterpret_cast<const float4_t*>(sp + n) : float4_t{0.f, 0.f, 0.f, 0.f};
  }
  const float* xcol = a.xbc + head * a.vdim + min(col, a.vdim - 1);
  const float* Bg = a.xbc + a.off_b + group * N;
  const float* Cg = a.xbc + a.off_c + group * N;
  const int chunks = (a.n + C - 1) / C;
  SsdOperands<NT> o;
  // channels past the state meet zeros of S, tokens past the end zeros of M and e (rows of Y are not stored)
  auto load_own = [&](int c) {
    const float* src = a.tm + ((int64_t)c * a.heads + head) * SsdChunk::floats;
#pragma unroll
    for (int k = 0; k < 4; ++k) {
      o.e[k] = *reinterpret_cast<const float4_t*>(src + SsdChunk::e + k * 16 + q4 * 4);
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int64_t row = (int64_t)min(c * C + k * 16 + q4 * 4 + i, a.n - 1) * a.ld;
        o.x[k][i] = xcol[row];
#pragma unroll
        for (int t = 0; t < NT; ++t) o.b[t][k][i] = Bg[row + min((wave * NT + t) * 16 + l16, N - 1)];
      }
      o.m[k] = *reinterpret_cast<const float4_t*>(src + SsdChunk::m + (wave * (wave + 1) / 2 + min(k, wave)) * 256 + lane * 4);
    }
    o.total = src[SsdChunk::p0 + C - 1];
  };
  auto load_read = [&](int c) {
    const float* cr = Cg + (int64_t)min(c * C + wave * 16 + l16, a.n - 1) * a.ld;
#pragma unroll
    for (int t = 0; t < 4 * NT; ++t) o.c[t] = *reinterpret_cast<const float4_t*>(cr + min(t * 16 + q4 * 4, N - 4));
    o.p0 = *reinterpret_cast<const float4_t*>(a.tm + ((int64_t)c * a.heads + head) * SsdChunk::floats + SsdChunk::p0 +
                                              wave * 16 + q4 * 4);
  };
  load_own(0);
  load_read(0);
  for (int c = 0; c < chunks; ++c) {
    const int par = c & 1, next = min(c + 1, chunks - 1);
#pragma unroll
    for (int t = 0; t < NT; ++t) state[par][wave * NT + t][lane] = S[t];
    // the next state needs only this wave's own part of the last one
#pragma unroll
    for (int t = 0; t < NT; ++t) S[t] *= o.total;
#pragma unroll
    for (int k = 0; k < 4; ++k)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const float xe = o.x[k][i] * o.e[k][i];
#pragma unroll
        for (int t = 0; t < NT; ++t) S[t] = __builtin_amdgcn_mfma_f32_16x16x4f32(o.b[t][k][i], xe, S[t], 0, 0, 0);
      }
    float4_t mx = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int k = 0; k < 4; ++k)
      if (k <= wave) {
#pragma unroll
        for (int i = 0; i < 4; ++i) mx = __builtin_amdgcn_mfma_f32_16x16x4f32(o.m[k][i], o.x[k][i], mx, 0, 0, 0);
      }
#pragma unroll
    for (int t = 0; t < NT; ++t)  // channels past the state stay zero
      if ((wave * NT + t) * 16 + q4 * 4 >= N) S[t] = float4_t{0.f, 0.f, 0.f, 0.f};
    load_own(next);
    __syncthreads();
    float4_t y[2];
    y[0] = y[1] = float4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int t = 0; t < 4 * NT; ++t) {
      const float4_t s = state[par][t][lane];
#pragma unroll
      for (int i = 0; i < 4; ++i) y[t & 1] = __builtin_amdgcn_mfma_f32_16x16x4f32(o.c[t][i], s[i], y[t & 1], 0, 0, 0);
    }
    const float4_t out = (y[0] + y[1]) * o.p0 + mx;
    load_read(next);
    const int t0 = c * C + wave * 16 + q4 * 4;
#pragma unroll
    for (int i = 0; i < 4; ++i)
      if (col_ok && t0 + i < a.n) a.y[(int64_t)(t0 + i) * a.ldy + head * a.vdim + col] = out[i];
  }
#pragma unroll
  for (int t = 0; t < NT; ++t) {
    const int n = (wave * NT + t) * 16 + q4 * 4;
    if (col_ok && n < N) *reinterpret_cast<float4_t*>(sp + n) = S[t];
  }
}

// One decode token.  A workgroup owns 16 columns of a head, a row of 16 lanes a column.  Grid: heads * ceil(vdim / 16).
using SsdStepArgs = dvSsdStepArgs;

template <int NT>
__global__ __launch_bounds__(256) void ssd_step_kernel(SsdStepArgs a) {
  const int head = blockIdx.x % a.heads, tile = blockIdx.x / a.heads;
  const int sub = threadIdx.x & 15, col = tile * kSsdCols + (threadIdx.x >> 4), N = a.state_s;
  const bool ok = col < a.vdim;
  const int at = head * a.vdim + min(col, a.vdim - 1), group = head / (a.heads / a.groups);
  float* sp = a.S + (int64_t)at * N;
  float4_t S[NT], B[NT], C[NT];
#pragma unroll
  for (int t = 0; t < NT; ++t) {
    const int n = min(t * 64 + sub * 4, N - 4);
    S[t] = *reinterpret_cast<const float4_t*>(sp + n);
    B[t] = *reinterpret_cast<const float4_t*>(a.p + a.off_b + group * N + n);
    C[t] = *reinterpret_cast<const float4_t*>(a.p + a.off_c + group * N + n);
  }
  const float x = a.p[at], z = a.p[a.off_z + at], D = a.D[head];
  const SsdGates g = ssd_gates(a.p[a.off_dt + head], a.dt_bias[head], a.A_log[head]);
  const float u = g.dt * x;
  float y = 0.f;
#pragma unroll
  for (int t = 0; t < NT; ++t)
    if (t * 64 + sub * 4 < N) {
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        S[t][i] = __builtin_fmaf(g.a, S[t][i], u * B[t][i]);
        y = __builtin_fmaf(S[t][i], C[t][i], y);
      }
      if (ok) *reinterpret_cast<float4_t*>(sp + t * 64 + sub * 4) = S[t];
    }
  y = row16_sum(y);
  if (ok && sub == 0) a.y[at] = (y + D * x) * silu_f(z);
}

}  // namespace dv
