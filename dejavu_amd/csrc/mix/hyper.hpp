// Several residual streams around the sublayers (fp32): every sublayer reads a weighted sum of them and its result is
// written back to all of them through a small matrix; the embedding that starts them; RMS norms of the rows in between.
#pragma once
#include "elem.hpp"

namespace dv {

using HyperArgs = dvHyper;

// coef: [streams] in, [streams] out, [streams][streams] mix.
__device__ __forceinline__ void hyper_coefficients(const HyperArgs& a, float* coef, int tid, int threads) {
  const int S = a.streams;
  for (int i = tid; i < S * (S + 2); i += threads)
    coef[i] = i < S ? (a.in ? a.in[i] : 0.f) : (i < 2 * S ? (a.out ? a.out[i - S] : 0.f) : (a.mix ? a.mix[i - 2 * S] : 0.f));
}

// One channel: the streams old[0 .. streams - 1] become the new ones at x (one every `width`); returns u.
template <int SM>
__device__ __forceinline__ float hyper_apply(const HyperArgs& a, const float* coef, float* x, const float (&old)[SM], float y) {
  const int S = a.streams;
  float u = 0.f;
  for (int t = 0; t < S; ++t) {
    float v = coef[S + t] * y;
#pragma unroll
    for (int s = 0; s < SM; ++s)
      if (s < S) v = __builtin_fmaf(coef[2 * S + s * S + t], old[s], v);
    x[(int64_t)t * a.width] = v;
    u = __builtin_fmaf(coef[t], v, u);
  }
  return u;
}

using EmbedArgs = dvEmbedArgs;
using RmsOut = dvRmsOut;

// One workgroup per token (several for one token without a norm: grid.y).  EMBED: the streams start with the embedding;
// else y joins them (null: they stay).  Four channels per thread; u is kept in LDS for the norm (dynamic, width floats).
// SM: streams kept in registers (>= streams).  TH: threads.
template <typename T, int SM, bool EMBED, int TH>
__global__ __launch_bounds__(TH) void hyper_rows_kernel(const T* __restrict__ y, HyperArgs a, EmbedArgs em, RmsOut norm) {
  extern __shared__ __attribute__((aligned(16))) unsigned char smem_raw[];
  float* us = reinterpret_cast<float*>(smem_raw);
  __shared__ float coef[SM * (SM + 2)], red[TH / 64];
  const int tid = threadIdx.x, S = a.streams;
  const int64_t row = blockIdx.x;
  float* x = a.x + row * S * a.width;
  const T *e0 = nullptr, *e1 = nullptr;
  if constexpr (EMBED) {
    const int64_t* tokens = reinterpret_cast<const int64_t*>(em.tokens);
    int64_t* history = reinterpret_cast<int64_t*>(em.history);
    const int64_t pos = seq_position(em.pos_dev, em.pos_host) + row, tok = tokens[row];
    if (tok >= 0 && tok < em.vocab) e0 = reinterpret_cast<const T*>(em.embed) + tok * a.width;
    if (em.bigram) {
      int64_t b = em.buckets;
      if (pos > 0) {
        const int64_t prev = row > 0 ? tokens[row - 1] : history[min(pos, em.capacity) - 1];
        b = (prev * em.mul_prev + tok * em.mul_cur) % em.buckets;
        if (b < 0) b += em.buckets;
      }
      e1 = reinterpret_cast<const T*>(em.bigram) + b * a.width;
    }
    if (tid == 0 && blockIdx.y == 0 && pos < em.capacity) history[pos] = tok;  // no workgroup of this call reads it
  }
  // the first values are requested before the coefficients are there
  float4_t old[SM], add[2];
  auto load = [&](int c) {
    if constexpr (EMBED) {
      add[0] = add[1] = float4_t{0.f, 0.f, 0.f, 0.f};
      if (e0) add[0] = load_quad(e0 + c);
      if (e1) add[1] = load_quad(e1 + c);
    } else {
#pragma unroll
      for (int s = 0; s < SM; ++s)
        if (s < S) old[s] = *reinterpret_cast<const float4_t*>(x + (int64_t)s * a.width + c);
      if (y) add[0] = load_quad(y + row * a.width + c);
    }
  };
  const int c0 = (blockIdx.y * TH + tid) * 4, step = gridDim.y * TH * 4;
  if (c0 < a.width) load(c0);
  hyper_coefficients(a, coef, tid, TH);
  __syncthreads();
  float ss = 0.f;
  for (int c = c0; c < a.width; c += step) {
    float4_t u = {0.f, 0.f, 0.f, 0.f};
    if (c != c0) load(c);
    if constexpr (EMBED) {
      const float4_t v = add[0] * em.scale + add[1];
      for (int s = 0; s < S; ++s) {
        *reinterpret_cast<float4_t*>(x + (int64_t)s * a.width + c) = v;
        u += v * coef[s];
      }
    } else {
      if (y) {
        for (int t = 0; t < S; ++t) {
          float4_t v = add[0] * coef[S + t];
#pragma unroll
          for (int s = 0; s < SM; ++s)
            if (s < S) v += old[s] * coef[2 * S + s * S + t];
          *reinterpret_cast<float4_t*>(x + (int64_t)t * a.width + c) = v;
          u += v * coef[t];
        }
      } else {
#pragma unroll
        for (int s = 0; s < SM; ++s)
          if (s < S) u += old[s] * coef[s];
      }
    }
    if (a.u) *reinterpret_cast<float4_t*>(a.u + row * a.width + c) = u;
    if (norm.h) {
      *reinterpret_cast<float4_t*>(us + c) = u;
#pragma unroll
      for (int e = 0; e < 4; ++e)
        if (c + e < norm.dim) ss = __builtin_fmaf(u[e], u[e], ss);
    }
  }
  if (!norm.h) return;  // the same for the whole grid
  ss = wave_sum(ss);
  if ((tid & 63) == 0) red[tid >> 6] = ss;
  __syncthreads();
  ss = 0.f;
#pragma unroll
  for (int i = 0; i < TH / 64; ++i) ss += red[i];
  const float s = 1.f / sqrtf(ss / norm.dim + norm.eps);
  T* h = reinterpret_cast<T*>(norm.h) + row * a.width;
  for (int c = c0; c < a.width; c += step)  // the entries this thread has written
    store_quad(h + c, *reinterpret_cast<const float4_t*>(us + c) * s * *reinterpret_cast<const float4_t*>(norm.w + c));
}

using HeadGroup = dvHeadGroup;
using HeadArgs = dvHeadArgs;

// The heads of a projection's rows: RMS-normed with a weight, or mixed with other rows.  A row of 16 lanes per (token,
// head); eight channels per lane at a time, the first 128 kept in registers.
template <typename T>
__global__ __launch_bounds__(256) void head_rows_kernel(HeadArgs a) {
  const int heads = a.g[0].heads + a.g[1].heads + a.g[2].heads;
  const unsigned unit = blockIdx.x * 16 + (threadIdx.x >> 4);
  const int sub = threadIdx.x & 15;
  const bool ok = unit < (unsigned)a.n * (unsigned)heads;  // whole rows of lanes: the sum below stays inside one
  const int64_t row = ok ? unit / (unsigned)heads : 0;
  int h = ok ? (int)(unit % (unsigned)heads) : 0, base = 0, gi = 0;
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
  const HeadGroup g = a.g[gi];
  const T* in = reinterpret_cast<const T*>(a.in) + row * a.ldi + base + (int64_t)h * g.stride;
  const T* other = g.other ? reinterpret_cast<const T*>(g.other) + row * g.ldo + (int64_t)h * g.stride : nullptr;
  T* out = reinterpret_cast<T*>(g.out) + row * g.ld + (int64_t)h * g.stride;
  const float lam = other ? *g.lambda : 0.f;
  Pack8<T> v, o0;
  Pack8<float> w0;
  v.zero();
  if (sub * 8 < g.stride) {
    v.load(in + sub * 8);
    if (g.w) w0.load(g.w + sub * 8);
    if (other) o0.load(other + sub * 8);
  }
  float ss = 0.f;
#pragma unroll
  for (int e = 0; e < 8; ++e) ss = __builtin_fmaf(v.get(e), v.get(e), ss);  // entries from dim on are zero
  for (int c = 128 + sub * 8; c < g.stride; c += 128) {
    Pack8<T> t;
    t.load(in + c);
#pragma unroll
    for (int e = 0; e < 8; ++e) ss = __builtin_fmaf(t.get(e), t.get(e), ss);
  }
  ss = row16_sum(ss);
  if (!ok) return;
  const float s = g.w ? 1.f / sqrtf(ss / g.dim + g.eps) : 1.f;
  for (int c = sub * 8; c < g.stride; c += 128) {
    Pack8<T> t = v;
    if (c >= 128) t.load(in + c);
    __attribute__((aligned(16))) T r[8];
    if (g.w) {
      Pack8<float> w = w0;
      if (c >= 128) w.load(g.w + c);
#pragma unroll
      for (int e = 0; e < 8; ++e) r[e] = from_f<T>(t.get(e) * s * w.get(e));
    } else if (other) {
      Pack8<T> o = o0;
      if (c >= 128) o.load(other + c);
#pragma unroll
      for (int e = 0; e < 8; ++e) r[e] = from_f<T>(__builtin_fmaf(lam, o.get(e), (1.f - lam) * t.get(e)));
    } else {
#pragma unroll
      for (int e = 0; e < 8; ++e) r[e] = from_f<T>(t.get(e));
    }
    *reinterpret_cast<Pack8<T>*>(out + c) = *reinterpret_cast<const Pack8<T>*>(r);
  }
}

// out = t / rms(t) * w per group of gs entries, t = y silu(z).  W waves per (row, group); VEC: gs % 4 == 0, four entries
// per thread at a time, the first NX packets kept in registers.  The entries from dim on become zero.
template <typename T, int W, bool VEC>
__global__ __launch_bounds__(256) void gated_group_norm_kernel(const float* __restrict__ y, int64_t ldy,
                                                               const T* __restrict__ z, int64_t ldz, int64_t rows,
                                                               int dim, int gs, int padded, const float* __restrict__ w,
                                                               float eps, T* __restrict__ out) {
  constexpr int TH = 64 * W, NX = 4, V = VEC ? 4 : 1;
  __shared__ float red[4];
  const int groups = dim / gs, t = threadIdx.x % TH;
  const unsigned unit = blockIdx.x * (4 / W) + threadIdx.x / TH;
  const bool ok = unit < rows * groups;  // whole waves
  const int64_t row = ok ? unit / (unsigned)groups : 0;
  const int g = ok ? (int)(unit % (unsigned)groups) : 0;
  const float* yr = y + row * ldy + g * gs;
  const T* zr = z + row * ldz + g * gs;
  auto value = [&](int c) {
    float4_t v = {0.f, 0.f, 0.f, 0.f};
    if constexpr (VEC) {
      v = *reinterpret_cast<const float4_t*>(yr + c);
      const float4_t k = load_quad(zr + c);
#pragma unroll
      for (int e = 0; e < 4; ++e) v[e] *= silu_f(k[e]);
    } else {
      v[0] = yr[c] * silu_f(to_f(zr[c]));
    }
    return v;
  };
  float4_t v[NX];
  float ss = 0.f;
  auto squares = [&](const float4_t& a) {
#pragma unroll
    for (int e = 0; e < V; ++e) ss = __builtin_fmaf(a[e], a[e], ss);
  };
#pragma unroll
  for (int i = 0; i < NX; ++i) {
    const int c = (i * TH + t) * V;
    v[i] = float4_t{0.f, 0.f, 0.f, 0.f};
    if (c < gs) v[i] = value(c);
    squares(v[i]);
  }
  for (int c = (NX * TH + t) * V; c < gs; c += TH * V) squares(value(c));
  ss = wave_sum(ss);
  if constexpr (W > 1) {
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = ss;
    __syncthreads();
    ss = 0.f;
#pragma unroll
    for (int i = 0; i < W; ++i) ss += red[threadIdx.x / TH * W + i];
  }
  if (!ok) return;
  const float s = 1.f / sqrtf(ss / gs + eps);
  T* o = out + row * padded + g * gs;
  const float* wr = w + g * gs;
  auto put = [&](const float4_t& a, int c) {
    if constexpr (VEC) store_quad(o + c, a * s * *reinterpret_cast<const float4_t*>(wr + c));
    else o[c] = from_f<T>(a[0] * s * wr[c]);
  };
#pragma unroll
  for (int i = 0; i < NX; ++i) {
    const int c = (i * TH + t) * V;
    if (c < gs) put(v[i], c);
  }
  for (int c = (NX * TH + t) * V; c < gs; c += TH * V) put(value(c), c);
  if (g == groups - 1)
    for (int c = dim + t; c < padded; c += TH) out[row * padded + c] = from_f<T>(0.f);
}

}  // namespace dv
