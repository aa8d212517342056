// Causal depthwise convolution over the tokens of a portion, with the last taps - 1 inputs of a sequence as state.
#pragma once
#include "elem.hpp"

namespace dv {

using ConvGroup = dvConvGroup;
using ConvArgs = dvConvArgs;

// A lane owns eight channels of one head and walks TB consecutive tokens with the last TAPS inputs in registers; the
// LPH lanes of a head (a power of two, 8 LPH >= stride) add up its norm.  Grid: (units of heads, token blocks).
constexpr int kConvTokens = 8;

template <int LPH>
__device__ __forceinline__ float lanes_sum(float v) {
  if constexpr (LPH >= 2) v = dpp_add<0xB1>(v);
  if constexpr (LPH >= 4) v = dpp_add<0x4E>(v);
  if constexpr (LPH >= 8) v = dpp_add<0x141>(v);
  if constexpr (LPH >= 16) v = dpp_add<0x140>(v);
  if constexpr (LPH >= 32) v += __shfl_xor(v, 16, kWave);
  if constexpr (LPH >= 64) v += __shfl_xor(v, 32, kWave);
  return v;
}

template <typename T, typename TO, int LPH, int TAPS>
__global__ __launch_bounds__(256) void short_conv_kernel(ConvArgs a) {
  constexpr int HPB = 256 / LPH;  // heads per workgroup
  const int heads = a.g[0].heads + a.g[1].heads + a.g[2].heads;
  const int unit = blockIdx.x * HPB + threadIdx.x / LPH, c0 = threadIdx.x % LPH * 8;
  int h = unit < heads ? unit : 0, base = 0, gi = 0;
  if (h >= a.g[0].heads) {
    h -= a.g[0].heads;
    base = a.g[0].heads * a.g[0].stride;
    gi = 1;
    if (h >= a.g[1].heads) {
      h -= a.g[1].heads;
      base += a.g[1].heads * a.g[1].stride;
      gi = 2;
    }
  }
  const ConvGroup g = a.g[gi];
  const bool on = unit < heads && c0 < g.stride;
  const int c = min(c0, g.stride - 8);
  const int ch = base + h * g.stride + c;
  const T* in = reinterpret_cast<const T*>(a.in) + ch;
  float w[TAPS][8], u[TAPS][8];
  {
    float4_t wv[TAPS * 2];  // eight channels x TAPS, contiguous
#pragma unroll
    for (int i = 0; i < TAPS * 2; ++i)
      wv[i] = *reinterpret_cast<const float4_t*>(a.w + (int64_t)ch * TAPS + i * 4);
#pragma unroll
    for (int e = 0; e < 8; ++e)
#pragma unroll
      for (int j = 0; j < TAPS; ++j) w[j][e] = wv[(e * TAPS + j) >> 2][(e * TAPS + j) & 3];
  }
  float bias[8];
#pragma unroll
  for (int e = 0; e < 8; ++e) bias[e] = a.b ? a.b[ch + e] : 0.f;
  const int t0 = blockIdx.y * kConvTokens, t1 = min(a.n, t0 + kConvTokens);
  Pack8<T> next[kConvTokens];
#pragma unroll
  for (int i = 0; i < kConvTokens; ++i) {
    next[i].load(in + (int64_t)min(t0 + i, t1 - 1) * a.ldi);
  }
#pragma unroll
  for (int j = 0; j < TAPS - 1; ++j) {  // the inputs before the block
    const int s = t0 - (TAPS - 1) + j;
    Pack8<T> v;
    v.load(in + (int64_t)max(s, 0) * a.ldi);
#pragma unroll
    for (int e = 0; e < 8; ++e) u[j][e] = v.get(e);
    if (s < 0) {
#pragma unroll
      for (int e = 0; e < 8; ++e) u[j][e] = a.state[(int64_t)(ch + e) * (TAPS - 1) + TAPS - 1 + s];
    }
  }
  TO* out = reinterpret_cast<TO*>(g.out) + (int64_t)h * g.stride + c;
#pragma unroll
  for (int i = 0; i < kConvTokens; ++i) {
    float y[8], ss = 0.f;
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      u[TAPS - 1][e] = next[i].get(e);
      float v = bias[e];
#pragma unroll
      for (int j = 0; j < TAPS; ++j) v = __builtin_fmaf(w[j][e], u[j][e], v);
      y[e] = a.silu ? silu_f(v) : v;
      if (c + e < g.dim) ss = __builtin_fmaf(y[e], y[e], ss);
    }
#pragma unroll
    for (int j = 0; j < TAPS - 1; ++j)
#pragma unroll
      for (int e = 0; e < 8; ++e) u[j][e] = u[j + 1][e];
    ss = lanes_sum<LPH>(on ? ss : 0.f);  // by every lane: the lanes of a head may share a wave with a group without norm
    const float s = g.norm == 1 ? 1.f / sqrtf(ss / g.dim + g.eps) : (g.norm == 2 ? g.scale / sqrtf(ss + 1e-6f) : 1.f);
#pragma unroll
    for (int e = 0; e < 8; ++e) y[e] *= s;
    if (on && t0 + i < t1) {
      __attribute__((aligned(16))) TO o[8];
#pragma unroll
      for (int e = 0; e < 8; ++e) o[e] = from_f<TO>(y[e]);
      *reinterpret_cast<Pack8<TO>*>(out + (int64_t)(t0 + i) * g.ld) = *reinterpret_cast<const Pack8<TO>*>(o);
    }
  }
}

// Any number of taps and any head size: one wave per (token, head), values computed twice where a norm needs them.
template <typename T, typename TO>
__global__ __launch_bounds__(256) void short_conv_any_kernel(ConvArgs a) {
  const int lane = threadIdx.x & 63;
  const int heads = a.g[0].heads + a.g[1].heads + a.g[2].heads;
  const int64_t task = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
  if (task >= (int64_t)a.n * heads) return;
  const int t = (int)(task / heads);
  int h = (int)(task % heads), base = 0, gi = 0;
  if (h >= a.g[0].heads) {
    h -= a.g[0].heads;
    base = a.g[0].heads * a.g[0].stride;
    gi = 1;
    if (h >= a.g[1].heads) {
      h -= a.g[1].heads;
      base += a.g[1].heads * a.g[1].stride;
      gi = 2;
    }
  }
  const ConvGroup g = a.g[gi];
  const T* in = reinterpret_cast<const T*>(a.in);
  base += h * g.stride;
  auto value = [&](int c) {
    const int ch = base + c;
    float y = a.b ? a.b[ch] : 0.f;
    for (int j = 0; j < a.taps; ++j) {
      const int s = t - (a.taps - 1) + j;
      const float u = s >= 0 ? to_f(in[s * a.ldi + ch]) : a.state[(int64_t)ch * (a.taps - 1) + a.taps - 1 + s];
      y = __builtin_fmaf(a.w[(int64_t)ch * a.taps + j], u, y);
    }
    return a.silu ? silu_f(y) : y;
  };
  float s = 1.f;
  if (g.norm) {
    float ss = 0.f;
    for (int c = lane; c < g.dim; c += 64) {
      const float v = value(c);
      ss = __builtin_fmaf(v, v, ss);
    }
    ss = wave_sum(ss);
    s = g.norm == 1 ? 1.f / sqrtf(ss / g.dim + g.eps) : g.scale / sqrtf(ss + 1e-6f);
  }
  TO* out = reinterpret_cast<TO*>(g.out) + (int64_t)t * g.ld + (int64_t)h * g.stride;
  for (int c = lane; c < g.stride; c += 64) out[c] = from_f<TO>(value(c) * s);
}

// state <- the last taps - 1 inputs of (state, in[0..n)).  One thread per channel; in place: a slot is written
// after every slot that is read later has a larger index.
template <typename T>
__global__ __launch_bounds__(256) void conv_state_kernel(const T* __restrict__ in, int64_t ldi, int n, int channels,
                                                         int taps, float* state) {
  const int ch = blockIdx.x * 256 + threadIdx.x;
  if (ch >= channels) return;
  float* st = state + (int64_t)ch * (taps - 1);
  for (int j = 0; j < taps - 1; ++j) {
    const int s = n - (taps - 1) + j;
    st[j] = s >= 0 ? to_f(in[(int64_t)s * ldi + ch]) : st[j + n];
  }
}

}  // namespace dv
