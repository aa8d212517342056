// Causal depthwise convolution over the tokens of a portion, with the last taps - 1 inputs of a sequence as state.
#pragma once
#include "elem.hpp"

namespace dv {

using ConvGroup = dvConvGroup;
using ConvArgs = dvConvArgs;

// One wave per (token, head); a lane holds up to NE channels.  TO: type of the outputs.
template <typename T, typename TO, int NE>
__global__ __launch_bounds__(256) void short_conv_kernel(ConvArgs a) {
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
  float v[NE], ss = 0.f;
#pragma unroll
  for (int i = 0; i < NE; ++i) {
    const int c = lane + i * 64;
    v[i] = 0.f;
    if (c < g.stride) {
      const int ch = base + c;
      float y = 0.f;
      for (int j = 0; j < a.taps; ++j) {
        const int s = t - (a.taps - 1) + j;
        const float u = s >= 0 ? to_f(in[s * a.ldi + ch]) : a.state[(int64_t)ch * (a.taps - 1) + a.taps - 1 + s];
        y = __builtin_fmaf(a.w[(int64_t)ch * a.taps + j], u, y);
      }
      v[i] = a.silu ? silu_f(y) : y;
      if (c < g.dim) ss = __builtin_fmaf(v[i], v[i], ss);
    }
  }
  float s = 1.f;
  if (g.norm) {
    ss = wave_sum(ss);
    s = g.norm == 1 ? 1.f / sqrtf(ss / g.dim + g.eps) : g.scale / sqrtf(ss + 1e-6f);
  }
  TO* out = reinterpret_cast<TO*>(g.out) + (int64_t)t * g.ld + (int64_t)h * g.stride;
#pragma unroll
  for (int i = 0; i < NE; ++i) {
    const int c = lane + i * 64;
    if (c < g.stride) out[c] = from_f<TO>(v[i] * s);
  }
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
