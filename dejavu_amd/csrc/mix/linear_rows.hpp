// One activation row times a weight matrix (the products of a decode step), with what comes before and after the
// product inside the launch:
//   before: nothing, an RMS norm of the row, a per-head RMS norm with an output gate, or an RMS norm per group;
//   after : plain store, a gated unit, a short convolution with its state, dynamic tanh + residual add + the next
//           dynamic tanh, or the update of several residual streams with the row that the next norm reads.
// A wave owns R consecutive rows of W at a time; the row x is staged in LDS once per workgroup.
#pragma once
#include "elem.hpp"
#include "hyper.hpp"
#include "stream.hpp"

namespace dv {

using RowsArgs = dvRowArgs;

// Short convolution of one channel's newest value with its state; returns the filtered value.
__device__ __forceinline__ float conv_step(float u, const float* __restrict__ w, float* __restrict__ st, int taps) {
  float y = w[taps - 1] * u;
  for (int j = 0; j < taps - 1; ++j) {
    const float old = st[j];
    y = __builtin_fmaf(w[j], old, y);
    if (j > 0) st[j - 1] = old;
  }
  if (taps > 1) st[taps - 2] = u;
  return y;
}

template <typename T, int BEFORE>
__device__ __forceinline__ void stage_row(const RowsArgs& a, T* xs, float* red) {
  const int tid = threadIdx.x, K = a.K;
  if constexpr (BEFORE == DV_ROW_PLAIN) {
    const T* x = reinterpret_cast<const T*>(a.x);
    for (int i = tid * 8; i < K; i += 4 * 2048) {  // four packets requested together
      Pack8<T> v[4];
#pragma unroll
      for (int u = 0; u < 4; ++u) v[u].load(x + min(i + u * 2048, K - 8));
#pragma unroll
      for (int u = 0; u < 4; ++u)
        if (i + u * 2048 < K) *reinterpret_cast<Pack8<T>*>(xs + i + u * 2048) = v[u];
    }
  } else if constexpr (BEFORE == DV_ROW_RMS) {
    const float* x = reinterpret_cast<const float*>(a.x);
    constexpr int NX = 4;  // packets of four values and weights a thread keeps; longer rows read the rest again
    float4_t v[NX], w[NX];
    float ss = 0.f;
#pragma unroll
    for (int u = 0; u < NX; ++u) {
      const int i = min(tid * 4 + u * 1024, K - 4);
      v[u] = *reinterpret_cast<const float4_t*>(x + i);
      w[u] = *reinterpret_cast<const float4_t*>(a.xw + i);
    }
    auto squares = [&](const float4_t& t, int i) {
#pragma unroll
      for (int e = 0; e < 4; ++e)
        if (i + e < a.norm_dim) ss = __builtin_fmaf(t[e], t[e], ss);
    };
#pragma unroll
    for (int u = 0; u < NX; ++u) squares(v[u], tid * 4 + u * 1024);
    for (int i = tid * 4 + NX * 1024; i < a.norm_dim; i += 1024) squares(*reinterpret_cast<const float4_t*>(x + i), i);
    ss = wave_sum(ss);
    if ((tid & 63) == 0) red[tid >> 6] = ss;
    __syncthreads();
    const float s = 1.f / sqrtf((red[0] + red[1] + red[2] + red[3]) / a.norm_dim + a.eps);
#pragma unroll
    for (int u = 0; u < NX; ++u)
      if (tid * 4 + u * 1024 < K) store_quad(xs + tid * 4 + u * 1024, v[u] * s * w[u]);
    for (int i = tid * 4 + NX * 1024; i < K; i += 1024)
      store_quad(xs + i, *reinterpret_cast<const float4_t*>(x + i) * s * *reinterpret_cast<const float4_t*>(a.xw + i));
  } else if constexpr (BEFORE == DV_ROW_GROUPS) {
    const float* x = reinterpret_cast<const float*>(a.x);
    const int gs = a.norm_dim;
    if (gs % 256 == 0 && a.x_dim <= 256 * 256) {
      // a wave's 256 consecutive entries lie in one group: sums per 256 entries, then per group
      __shared__ float part[256];
      constexpr int NX = 8;
      float4_t v[NX];
#pragma unroll
      for (int u = 0; u < NX; ++u) v[u] = *reinterpret_cast<const float4_t*>(x + min(tid * 4 + u * 1024, a.x_dim - 4));
      auto squares = [&](const float4_t& t, int i) {
        const float ss = wave_sum((t[0] * t[0] + t[1] * t[1]) + (t[2] * t[2] + t[3] * t[3]));
        if ((tid & 63) == 0) part[i >> 8] = ss;
      };
#pragma unroll
      for (int u = 0; u < NX; ++u)
        if (tid * 4 + u * 1024 < a.x_dim) squares(v[u], tid * 4 + u * 1024);  // x_dim % 256 == 0: whole waves
      for (int i = tid * 4 + NX * 1024; i < a.x_dim; i += 1024) squares(*reinterpret_cast<const float4_t*>(x + i), i);
      __syncthreads();
      auto put = [&](const float4_t& t, int i) {
        const int g = i / gs;
        float ss = 0.f;
        for (int p = g * (gs >> 8); p < (g + 1) * (gs >> 8); ++p) ss += part[p];
        store_quad(xs + i, t * (1.f / sqrtf(ss / gs + a.eps)) * *reinterpret_cast<const float4_t*>(a.xw + i));
      };
#pragma unroll
      for (int u = 0; u < NX; ++u)
        if (tid * 4 + u * 1024 < a.x_dim) put(v[u], tid * 4 + u * 1024);
      for (int i = tid * 4 + NX * 1024; i < a.x_dim; i += 1024) put(*reinterpret_cast<const float4_t*>(x + i), i);
    } else {  // a wave per group
      const int lane = tid & 63;
      for (int g = tid >> 6; g * gs < a.x_dim; g += 4) {
        float ss = 0.f;
        for (int c = lane; c < gs; c += 64) ss = __builtin_fmaf(x[g * gs + c], x[g * gs + c], ss);
        const float s = 1.f / sqrtf(wave_sum(ss) / gs + a.eps);
        for (int c = lane; c < gs; c += 64) xs[g * gs + c] = from_f<T>(x[g * gs + c] * s * a.xw[g * gs + c]);
      }
    }
    for (int i = a.x_dim + tid; i < K; i += 256) xs[i] = from_f<T>(0.f);
  } else {
    // a row of 16 lanes per head; eight channels per lane at a time, the first 128 kept in registers
    const float* x = reinterpret_cast<const float*>(a.x);
    const int heads = K / a.head_stride, sub = tid & 15;
    for (int h = tid >> 4; h < heads; h += 16) {
      const float* xh = x + (int64_t)h * a.head_stride;
      const float* gh = a.gate + (int64_t)h * a.head_stride;
      Pack8<float> v;
      v.zero();
      if (sub * 8 < a.head_stride) v.load(xh + sub * 8);
      float ss = 0.f;
#pragma unroll
      for (int e = 0; e < 8; ++e) ss = __builtin_fmaf(v.get(e), v.get(e), ss);
      for (int c = 128 + sub * 8; c < a.head_stride; c += 128) {
        Pack8<float> u;
        u.load(xh + c);
#pragma unroll
        for (int e = 0; e < 8; ++e) ss = __builtin_fmaf(u.get(e), u.get(e), ss);
      }
      const float s = 1.f / sqrtf(row16_sum(ss) / a.norm_dim + a.eps);
      for (int c = sub * 8; c < a.head_stride; c += 128) {
        Pack8<float> u = v, g;
        if (c >= 128) u.load(xh + c);
        g.load(gh + c);
#pragma unroll
        for (int e = 0; e < 8; ++e) xs[h * a.head_stride + c + e] = from_f<T>(u.get(e) * s * a.xw[c + e] * g.get(e));
      }
    }
  }
  __syncthreads();
}

template <typename T, int BEFORE, int AFTER, int R, int U>
__global__ __launch_bounds__(256) void linear_rows_kernel(RowsArgs a) {
  extern __shared__ __attribute__((aligned(16))) unsigned char smem_raw[];
  T* xs = reinterpret_cast<T*>(smem_raw);
  __shared__ float red[4];
  const int lane = threadIdx.x & 63;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  int nblocks = gridDim.x;
  if (a.side_x) {
    --nblocks;
    if ((int)blockIdx.x == nblocks) {
      float ss = 0.f;
      for (int i = threadIdx.x; i < a.side_dim; i += 256) ss = __builtin_fmaf(a.side_x[i], a.side_x[i], ss);
      ss = wave_sum(ss);
      if (lane == 0) red[wave] = ss;
      __syncthreads();
      const float s = 1.f / sqrtf((red[0] + red[1] + red[2] + red[3]) / a.side_dim + a.eps);
      T* o = reinterpret_cast<T*>(a.side_out) + (int64_t)seq_position(a.pos_dev, a.pos_host) * a.side_ld;
      for (int i = threadIdx.x; i < a.side_padded; i += 256) o[i] = from_f<T>(a.side_x[i] * s * a.side_w[i]);
      return;
    }
  }
  constexpr int CH = 8 * kWave;
  const T* W = reinterpret_cast<const T*>(a.W);
  const int K = a.K, ntasks = (a.M + R - 1) / R;
  int t = blockIdx.x * 4 + wave;
  Pack8<T> w[U][R];
  const T* wr[R];
  auto rows_of = [&](int task) {
#pragma unroll
    for (int r = 0; r < R; ++r) {
      const int row = task * R + r;
      wr[r] = W + (int64_t)(row < a.M ? row : 0) * a.ldw;
    }
  };
  auto load_w = [&](int base) {
#pragma unroll
    for (int u = 0; u < U; ++u)
#pragma unroll
      for (int r = 0; r < R; ++r) {
        w[u][r].load_stream(wr[r] + min(base + u * CH + lane * 8, K - 8));
      }
  };
  if (t < ntasks) {  // the first weights are requested before x is there
    rows_of(t);
    load_w(0);
  }
  __shared__ float coef[DV_HYPER_ROW_MAX * (DV_HYPER_ROW_MAX + 2)];
  if constexpr (AFTER == DV_OUT_HYPER) hyper_coefficients(a.hyper, coef, threadIdx.x, 256);
  stage_row<T, BEFORE>(a, xs, red);
  for (; t < ntasks; t += nblocks * 4) {
    // what the epilogue adds to is requested before the products
    float old[DV_HYPER_ROW_MAX], bias = 0.f;
    if constexpr (AFTER != DV_OUT_GLU) {
      const int row = min(t * R + min(lane, R - 1), a.M - 1);
      if (a.bias) bias = to_f(reinterpret_cast<const T*>(a.bias)[row]);
      if constexpr (AFTER == DV_OUT_HYPER) {
#pragma unroll
        for (int s = 0; s < DV_HYPER_ROW_MAX; ++s)
          old[s] = a.hyper.x[(int64_t)min(s, a.hyper.streams - 1) * a.hyper.width + row];
      }
    }
    float acc[R];
#pragma unroll
    for (int r = 0; r < R; ++r) acc[r] = 0.f;
    for (int base = 0; base < K; base += U * CH) {
#pragma unroll
      for (int u = 0; u < U; ++u) {
        const int k = base + u * CH + lane * 8;
        if (k < K) {
          Pack8<T> xv;
          xv = *reinterpret_cast<const Pack8<T>*>(xs + k);
#pragma unroll
          for (int r = 0; r < R; ++r)
#pragma unroll
            for (int e = 0; e < 8; ++e) acc[r] = __builtin_fmaf(w[u][r].get(e), xv.get(e), acc[r]);
        }
      }
      if (base + U * CH < K) load_w(base + U * CH);
    }
#pragma unroll
    for (int r = 0; r < R; ++r) acc[r] = wave_sum(acc[r]);
    const int row0 = t * R;
    if (t + nblocks * 4 < ntasks) {
      rows_of(t + nblocks * 4);
      load_w(0);
    }
    if constexpr (AFTER == DV_OUT_GLU) {
      static_assert(R % 2 == 0, "gate / up rows come in pairs");
#pragma unroll
      for (int r = 0; r < R; r += 2)
        if (lane == r && row0 + r + 1 < a.M)
          reinterpret_cast<T*>(a.out)[(row0 + r) >> 1] = from_f<T>(glu_f(acc[r], acc[r + 1], a.act, a.limit));
    } else {
      float v = 0.f;
#pragma unroll
      for (int r = 0; r < R; ++r)
        if (lane == r) v = acc[r];
      v += bias;
      const int row = row0 + lane;
      if (lane < R && row < a.M) {
        if constexpr (AFTER == DV_OUT_F32) {
          reinterpret_cast<float*>(a.out)[row] = v;
        } else if constexpr (AFTER == DV_OUT_T) {
          reinterpret_cast<T*>(a.out)[row] = from_f<T>(v);
        } else if constexpr (AFTER == DV_OUT_CONV) {
          if (row < a.conv_rows) {
            v = conv_step(v, a.conv_w + (int64_t)row * a.taps, a.conv_state + (int64_t)row * (a.taps - 1), a.taps);
            if (a.conv_b) v += a.conv_b[row];
            if (a.silu) v = silu_f(v);
          }
          reinterpret_cast<float*>(a.out)[row] = v;
        } else if constexpr (AFTER == DV_OUT_HYPER) {
          const float u = hyper_apply<DV_HYPER_ROW_MAX>(a.hyper, coef, a.hyper.x + row, old, v);
          if (a.hyper.u) a.hyper.u[row] = u;
        } else {
          residual_apply<T>(a.res, row, row, v);
        }
      }
    }
  }
}

}  // namespace dv
