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

// Chunk after chunk for 16 TC columns of a head.  Wave w owns channels [16 NT w, 16 NT (w + 1)) of the state as
// accumulators of the 16x16x4 products: row r of tile t is channel NT r + t of them, column l of tile c is column
// TC l + c, so that a lane's operands of all tiles lie side by side in memory.  Element i of a lane is row 4 (lane / 16) +
// i, which is also the operand layout of the product with C when its channels are taken in that order; the waves exchange
// the state through LDS once per chunk, then every wave makes 16 tokens of Y and its own channels of the next state.
// Operands are loaded by the lanes that use them, a chunk ahead; there are at most 63 loads per chunk, what the counter of
// outstanding loads holds.
template <int NT, int TC>
struct SsdOperands {
  float c[4][4 * NT];  // by owner of the channels: element NT i + t is step i of tile t
  float b[4][4][NT], x[4][4][TC];
  float4_t p0, m[4], e[4];
  float total;
};

template <int W>
__device__ __forceinline__ void load_floats(float* dst, const float* __restrict__ p) {
  typedef float vec_t __attribute__((ext_vector_type(W), aligned(4)));
  if constexpr (W == 1) {
    dst[0] = *p;
  } else {
    const vec_t v = *reinterpret_cast<const vec_t*>(p);
#pragma unroll
    for (int i = 0; i < W; ++i) dst[i] = v[i];
  }
}

// Grid: heads * ceil(vdim / (16 TC)).  Workgroups go to the eight XCDs in turn: neighbouring heads, which share B and C,
// are kept on one of them when heads % 8 == 0.  vdim % TC == 0.
template <int NT, int TC>
__global__ __launch_bounds__(256) void ssd_scan_kernel(SsdArgs a) {
  static_assert(NT == 1 || NT == 2 || NT == 4, "a lane's channels are one aligned load");
  constexpr int C = kSsdChunk;
  __shared__ __attribute__((aligned(16))) float4_t state[2][TC][4 * NT][64];
  const int xcds = a.heads % 8 == 0 ? 8 : 1, per = a.heads / xcds, item = blockIdx.x / xcds;
  const int head = blockIdx.x % xcds * per + item % per, tile = item / per;
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int l16 = lane & 15, q4 = lane >> 4, N = a.state_s;
  const int group = head / (a.heads / a.groups);
  const int col = (tile * kSsdCols + l16) * TC;
  const bool col_ok = col < a.vdim;
  const bool part = N != 64 * NT;  // some channels are not there
  const int n0 = (wave * 16 + q4 * 4) * NT;  // channel n0 + NT i + t is element i of tile t
  float* sp = a.S + ((int64_t)head * a.vdim + (col_ok ? col : 0)) * N;
  float4_t S[TC][NT];
#pragma unroll
  for (int c = 0; c < TC; ++c)
#pragma unroll
    for (int t = 0; t < NT; ++t)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int n = n0 + i * NT + t;
        S[c][t][i] = col_ok && n < N ? sp[c * N + n] : 0.f;
      }
  const int chunks = (a.n + C - 1) / C;
  // A load is a uniform address (on the scalar unit) plus what this lane adds to it in every chunk, in bytes.
  auto at = [](const float* base, unsigned bytes) {
    return reinterpret_cast<const float*>(reinterpret_cast<const char*>(base) + bytes);
  };
  const unsigned row4 = 4 * (unsigned)a.ld;
  const unsigned xoff = q4 * 4 * row4 + 4 * (unsigned)min(col, a.vdim - TC);
  const unsigned boff = q4 * 4 * row4 + 4 * (unsigned)min((wave * 16 + l16) * NT, N - NT);
  unsigned coff[4][NT];
#pragma unroll
  for (int w = 0; w < 4; ++w)
#pragma unroll
    for (int u = 0; u < NT; ++u) coff[w][u] = l16 * row4 + 4 * (unsigned)min((w * 16 + q4 * 4) * NT + u * 4, N - 4);
  const float* Xh = a.xbc + head * a.vdim;
  const float* Bg = a.xbc + a.off_b + group * N;
  const float* Cg = a.xbc + a.off_c + group * N + (int64_t)wave * 16 * a.ld;
  const unsigned yoff = q4 * 16 * (unsigned)a.ldy + 4 * col;
  // channels past the state meet zeros of S, tokens past the end zeros of M and e (rows of Y are not stored)
  auto load_xb = [&](SsdOperands<NT, TC>& o, int c, int k, int i) {
    const int64_t row = ((int64_t)c * C + k * 16 + i) * a.ld;
    load_floats<TC>(o.x[k][i], at(Xh + row, xoff));
    load_floats<NT>(o.b[k][i], at(Bg + row, boff));
  };
  auto load_c = [&](SsdOperands<NT, TC>& o, int c, int w, int u) {
    load_floats<4>(&o.c[w][u * 4], at(Cg + (int64_t)c * C * a.ld, coff[w][u]));
  };
  auto load_me = [&](SsdOperands<NT, TC>& o, int c, int k) {
    const float* src = a.tm + ((int64_t)c * a.heads + head) * SsdChunk::floats;
    o.m[k] = *reinterpret_cast<const float4_t*>(
        at(src + SsdChunk::m + (wave * (wave + 1) / 2 + min(k, wave)) * 256, lane * 16));
    o.e[k] = *reinterpret_cast<const float4_t*>(at(src + SsdChunk::e + k * 16, q4 * 16));
    if (k == 0) {
      o.p0 = *reinterpret_cast<const float4_t*>(at(src + SsdChunk::p0 + wave * 16, q4 * 16));
      o.total = src[SsdChunk::p0 + C - 1];
    }
  };
  // One chunk; the loads of chunk `next` are spread between the products, so that issuing them does not hold those up.
  auto step = [&](const SsdOperands<NT, TC>& o, SsdOperands<NT, TC>& x, int ch, int next, int par) {
    // the next state needs only this wave's own part of the last one
#pragma unroll
    for (int c = 0; c < TC; ++c)
#pragma unroll
      for (int t = 0; t < NT; ++t) {
        state[par][c][wave * NT + t][lane] = S[c][t];
        S[c][t] *= o.total;
      }
    float4_t mx[TC];
#pragma unroll
    for (int c = 0; c < TC; ++c) mx[c] = float4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int k = 0; k < 4; ++k)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
#pragma unroll
        for (int c = 0; c < TC; ++c) {
          const float xe = o.x[k][i][c] * o.e[k][i];
#pragma unroll
          for (int t = 0; t < NT; ++t)
            S[c][t] = __builtin_amdgcn_mfma_f32_16x16x4f32(o.b[k][i][t], xe, S[c][t], 0, 0, 0);
        }
        load_xb(x, next, k, i);
        __builtin_amdgcn_sched_group_barrier(0x008, TC * NT, 0);  // matrix instructions
        __builtin_amdgcn_sched_group_barrier(0x020, 2, 0);        // loads
      }
#pragma unroll
    for (int k = 0; k < 4; ++k)
      if (k <= wave) {
#pragma unroll
        for (int i = 0; i < 4; ++i)
#pragma unroll
          for (int c = 0; c < TC; ++c)
            mx[c] = __builtin_amdgcn_mfma_f32_16x16x4f32(o.m[k][i], o.x[k][i][c], mx[c], 0, 0, 0);
      }
    if (part) {  // channels past the state stay zero
#pragma unroll
      for (int c = 0; c < TC; ++c)
#pragma unroll
        for (int t = 0; t < NT; ++t)
#pragma unroll
          for (int i = 0; i < 4; ++i) S[c][t][i] = n0 + i * NT + t < N ? S[c][t][i] : 0.f;
    }
    __syncthreads();
    float4_t y[TC];
#pragma unroll
    for (int c = 0; c < TC; ++c) y[c] = float4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int w = 0; w < 4; ++w)
#pragma unroll
      for (int t = 0; t < NT; ++t) {
        float4_t s[TC];
#pragma unroll
        for (int c = 0; c < TC; ++c) s[c] = state[par][c][w * NT + t][lane];
#pragma unroll
        for (int i = 0; i < 4; ++i)
#pragma unroll
          for (int c = 0; c < TC; ++c)
            y[c] = __builtin_amdgcn_mfma_f32_16x16x4f32(o.c[w][i * NT + t], s[c][i], y[c], 0, 0, 0);
        load_c(x, next, w, t);
        if (t == 0) load_me(x, next, w);
        __builtin_amdgcn_sched_group_barrier(0x008, TC * 4, 0);
        __builtin_amdgcn_sched_group_barrier(0x020, 1, 0);
        if (t == 0) __builtin_amdgcn_sched_group_barrier(0x020, 2, 0);
      }
#pragma unroll
    for (int c = 0; c < TC; ++c) y[c] = y[c] * o.p0 + mx[c];
    const int t0 = ch * C + wave * 16;
#pragma unroll
    for (int i = 0; i < 4; ++i)
      if (col_ok && t0 + q4 * 4 + i < a.n) {
        float* yp = const_cast<float*>(at(a.y + (int64_t)(t0 + i) * a.ldy + head * a.vdim, yoff));
        if constexpr (TC == 2) {
          typedef float vec_t __attribute__((ext_vector_type(2), aligned(4)));
          *reinterpret_cast<vec_t*>(yp) = vec_t{y[0][i], y[1][i]};
        } else {
          *yp = y[0][i];
        }
      }
  };
  SsdOperands<NT, TC> even, odd;
#pragma unroll
  for (int k = 0; k < 4; ++k) {
#pragma unroll
    for (int i = 0; i < 4; ++i) load_xb(even, 0, k, i);
#pragma unroll
    for (int u = 0; u < NT; ++u) load_c(even, 0, k, u);
    load_me(even, 0, k);
  }
  for (int c = 0; c < chunks; c += 2) {
    step(even, odd, c, min(c + 1, chunks - 1), 0);
    if (c + 1 < chunks) step(odd, even, c + 1, min(c + 2, chunks - 1), 1);
  }
#pragma unroll
  for (int c = 0; c < TC; ++c)
#pragma unroll
    for (int t = 0; t < NT; ++t)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int n = n0 + i * NT + t;
        if (col_ok && n < N) sp[c * N + n] = S[c][t][i];
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
