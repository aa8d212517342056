// Products of a few rows (2..64 per workgroup column) with a bf16 weight on the matrix cores, with the epilogues of
// linear_rows.hpp.  The weight is the stream: a workgroup owns 32 rows of W, its four waves take every fourth
// 128-column chunk of K for all activation rows and add up in LDS.  Activations come through L1 / L2.
#pragma once
#include "elem.hpp"
#include "stream.hpp"

namespace dv {

using TileArgs = dvTileArgs;

// NT: tiles of 16 activation rows.  Grid: (ceil(M / 32), ceil(n / (16 NT))).
template <int AFTER, int NT>
__global__ __launch_bounds__(256) void linear_tiles_kernel(TileArgs a) {
  constexpr int RT = 2, U = 4;  // tiles of W rows; 32-column steps per chunk
  __shared__ __attribute__((aligned(16))) float4_t red[3][RT * NT][64];
  const int lane = threadIdx.x & 63;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int r16 = lane & 15, kq = (lane >> 4) * 8;
  const int m0 = blockIdx.x * 32, n0 = blockIdx.y * 16 * NT;
  const bf16_t* W = reinterpret_cast<const bf16_t*>(a.W);
  const bf16_t* X = reinterpret_cast<const bf16_t*>(a.x);
  const bf16_t* wp[RT];
  const bf16_t* xp[NT];
#pragma unroll
  for (int i = 0; i < RT; ++i) {
    const int m = m0 + i * 16 + r16;
    wp[i] = W + (int64_t)(m < a.M ? m : 0) * a.ldw;
  }
#pragma unroll
  for (int i = 0; i < NT; ++i) {
    const int n = n0 + i * 16 + r16;
    xp[i] = X + (int64_t)(n < a.n ? n : 0) * a.ldx;
  }
  float4_t acc[RT][NT];
#pragma unroll
  for (int i = 0; i < RT; ++i)
#pragma unroll
    for (int j = 0; j < NT; ++j) acc[i][j] = float4_t{0.f, 0.f, 0.f, 0.f};
  for (int k0 = wave * 32 * U; k0 < a.K; k0 += 4 * 32 * U) {
    Pack8<bf16_t> w[U][RT], x[U][NT];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int k = min(k0 + u * 32 + kq, a.K - 8);
#pragma unroll
      for (int i = 0; i < RT; ++i) w[u][i].load(wp[i] + k);
#pragma unroll
      for (int j = 0; j < NT; ++j) x[u][j].load(xp[j] + k);
    }
    if (k0 + 32 * U > a.K) {  // past the end of the rows
#pragma unroll
      for (int u = 0; u < U; ++u)
#pragma unroll
        for (int j = 0; j < NT; ++j)
          if (k0 + u * 32 + kq >= a.K) {
#pragma unroll
            for (int e = 0; e < 4; ++e) x[u][j].v[e] = 0u;
          }
    }
#pragma unroll
    for (int u = 0; u < U; ++u)
#pragma unroll
      for (int i = 0; i < RT; ++i)
#pragma unroll
        for (int j = 0; j < NT; ++j)
          acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, w[u][i].v),
                                                              __builtin_bit_cast(bf16x8_t, x[u][j].v), acc[i][j], 0, 0, 0);
  }
  if (wave > 0) {
#pragma unroll
    for (int i = 0; i < RT; ++i)
#pragma unroll
      for (int j = 0; j < NT; ++j) red[wave - 1][i * NT + j][lane] = acc[i][j];
  }
  __syncthreads();
  if (wave == 0) {
#pragma unroll
    for (int i = 0; i < RT; ++i)
#pragma unroll
      for (int j = 0; j < NT; ++j) {
        const float4_t t = acc[i][j] + ((red[0][i * NT + j][lane] + red[1][i * NT + j][lane]) + red[2][i * NT + j][lane]);
        red[0][i * NT + j][lane] = t;
      }
  }
  __syncthreads();
  for (int q = threadIdx.x; q < RT * NT * 64; q += 256) {
    const int tile = q >> 6, ln = q & 63;
    const int m = m0 + (tile / NT) * 16 + (ln >> 4) * 4, n = n0 + (tile % NT) * 16 + (ln & 15);
    if (n >= a.n) continue;
    float4_t v = red[0][tile][ln];
    if (AFTER != DV_OUT_GLU && a.bias) {
#pragma unroll
      for (int e = 0; e < 4; ++e) v[e] += to_f(reinterpret_cast<const bf16_t*>(a.bias)[min(m + e, a.M - 1)]);
    }
    if constexpr (AFTER == DV_OUT_GLU) {
#pragma unroll
      for (int e = 0; e < 4; e += 2)
        if (m + e + 1 < a.M)
          reinterpret_cast<bf16_t*>(a.out)[(int64_t)n * a.ldo + ((m + e) >> 1)] = (bf16_t)glu_f(v[e], v[e + 1], a.act, a.limit);
    } else {
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        if (m + e < a.M) {
          if constexpr (AFTER == DV_OUT_F32) reinterpret_cast<float*>(a.out)[(int64_t)n * a.ldo + m + e] = v[e];
          else if constexpr (AFTER == DV_OUT_T) reinterpret_cast<bf16_t*>(a.out)[(int64_t)n * a.ldo + m + e] = (bf16_t)v[e];
          else residual_apply<bf16_t>(a.res, (int64_t)n * a.M + m + e, m + e, v[e]);
        }
      }
    }
  }
}

}  // namespace dv
