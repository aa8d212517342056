// Elementwise kernels around the fp32 residual stream: embedding, dynamic tanh, gated feed-forward activation.
#pragma once
#include "elem.hpp"

namespace dv {

// x = x0 = embed[token]; h = norm(x).  Eight channels per thread; grid (tokens, ceil(width / 2048)).
template <typename T>
__global__ __launch_bounds__(256) void embed_norm_kernel(const int64_t* __restrict__ tokens, int64_t vocab,
                                                         const T* __restrict__ embed, int width, float* __restrict__ x,
                                                         float* __restrict__ x0, DynTanh norm, T* __restrict__ h) {
  const int64_t i = blockIdx.x;
  const int c = (blockIdx.y * 256 + threadIdx.x) * 8;
  if (c >= width) return;
  const int64_t tok = tokens[i];
  Pack8<T> v;
  if (tok >= 0 && tok < vocab) v.load(embed + tok * width + c);
  else v.zero();
  Pack8<float> f;
  __attribute__((aligned(16))) T o[8];
#pragma unroll
  for (int e = 0; e < 8; ++e) {
    const float t = v.get(e);
    if (e < 4) f.a[e] = t;
    else f.b[e - 4] = t;
    o[e] = from_f<T>(dyn_tanh(t, norm, c + e));
  }
  *reinterpret_cast<Pack8<float>*>(x + i * width + c) = f;
  if (x0) *reinterpret_cast<Pack8<float>*>(x0 + i * width + c) = f;
  *reinterpret_cast<Pack8<T>*>(h + i * width + c) = *reinterpret_cast<const Pack8<T>*>(o);
}

using ResidualArgs = dvResidual;
// What follows a sublayer's last product, for one value y of channel c.
template <typename T>
__device__ __forceinline__ void residual_apply(const ResidualArgs& a, int64_t at, int c, float y) {
  float v = a.x[at];
  v += dyn_tanh(y, a.post, c);
  if (a.x0) v += a.x0[at];
  a.x[at] = v;
  if (a.h) reinterpret_cast<T*>(a.h)[at] = from_f<T>(dyn_tanh(v, a.pre, c));
}

// y == nullptr: only x += x0 and h = pre(x).  Four channels per thread (width % 4 == 0).
template <typename T>
__global__ __launch_bounds__(256) void residual_norm_kernel(const T* __restrict__ y, int64_t quads, int width,
                                                            ResidualArgs a) {
  typedef T quad_t __attribute__((ext_vector_type(4)));
  for (int64_t q = (int64_t)blockIdx.x * 256 + threadIdx.x; q < quads; q += (int64_t)gridDim.x * 256) {
    const int64_t at = q * 4;
    const int c = (int)(at % width);
    float4_t v = *reinterpret_cast<const float4_t*>(a.x + at);
    if (y) {
      const quad_t u = *reinterpret_cast<const quad_t*>(y + at);
      const float4_t w = *reinterpret_cast<const float4_t*>(a.post.w + c), b = *reinterpret_cast<const float4_t*>(a.post.b + c);
#pragma unroll
      for (int e = 0; e < 4; ++e) v[e] += __builtin_fmaf(tanh_f(a.post.alpha * to_f(u[e])), w[e], b[e]);
    }
    if (a.x0) v += *reinterpret_cast<const float4_t*>(a.x0 + at);
    *reinterpret_cast<float4_t*>(a.x + at) = v;
    if (a.h) {
      const float4_t w = *reinterpret_cast<const float4_t*>(a.pre.w + c), b = *reinterpret_cast<const float4_t*>(a.pre.b + c);
      quad_t h;
#pragma unroll
      for (int e = 0; e < 4; ++e) h[e] = from_f<T>(__builtin_fmaf(tanh_f(a.pre.alpha * v[e]), w[e], b[e]));
      *reinterpret_cast<quad_t*>(reinterpret_cast<T*>(a.h) + at) = h;
    }
  }
}

// Clamped gated unit of one (gate, up) pair.
__device__ __forceinline__ float clamped_glu_f(float g, float u, float limit) {
  g = fminf(g, limit);
  u = fminf(fmaxf(u, -limit), limit);
  return g * sigmoid_f(1.702f * g) * (u + 1.f);
}

__device__ __forceinline__ float glu_f(float g, float u, int act, float limit) {
  return act == DV_GLU_RELU ? fmaxf(g, 0.f) * u : clamped_glu_f(g, u, limit);
}

// y[i] from gu[2 i] (gate) and gu[2 i + 1] (up); four outputs per thread, count % 4 == 0.
template <typename T, int ACT>
__global__ __launch_bounds__(256) void glu_kernel(const T* __restrict__ gu, int64_t count, float limit,
                                                  T* __restrict__ y) {
  const int64_t i = ((int64_t)blockIdx.x * 256 + threadIdx.x) * 4;
  if (i >= count) return;
  Pack8<T> v;
  v.load(gu + 2 * i);
#pragma unroll
  for (int e = 0; e < 4; ++e) y[i + e] = from_f<T>(glu_f(v.get(2 * e), v.get(2 * e + 1), ACT, limit));
}

// y = x / sqrt(mean(x^2) + eps) * w, the mean over the first `dim` entries (those up to `padded`, a multiple of 8, are
// zero).  One wave per row, eight entries per lane at a time.
template <typename T>
__global__ __launch_bounds__(256) void rms_rows_kernel(const T* __restrict__ x, int64_t ldx, int64_t rows, int dim,
                                                       int padded, const float* __restrict__ w, float eps,
                                                       T* __restrict__ y, int64_t ldy) {
  constexpr int NP = 4;  // packets a lane keeps; longer rows read the rest twice
  const int64_t r = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
  if (r >= rows) return;
  const int lane = threadIdx.x & 63;
  const T* xr = x + r * ldx;
  Pack8<T> v[NP];
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < NP; ++i) {
    const int c = (i * 64 + lane) * 8;
    if (c < padded) v[i].load(xr + c);
    else v[i].zero();
#pragma unroll
    for (int e = 0; e < 8; ++e) ss = __builtin_fmaf(v[i].get(e), v[i].get(e), ss);
  }
  for (int c = (NP * 64 + lane) * 8; c < padded; c += 512) {
    Pack8<T> t;
    t.load(xr + c);
#pragma unroll
    for (int e = 0; e < 8; ++e) ss = __builtin_fmaf(t.get(e), t.get(e), ss);
  }
  const float s = 1.f / sqrtf(wave_sum(ss) / dim + eps);
  auto put = [&](const Pack8<T>& t, int c) {
    __attribute__((aligned(16))) T o[8];
#pragma unroll
    for (int e = 0; e < 8; ++e) o[e] = from_f<T>(t.get(e) * s * w[c + e]);
    *reinterpret_cast<Pack8<T>*>(y + r * ldy + c) = *reinterpret_cast<const Pack8<T>*>(o);
  };
#pragma unroll
  for (int i = 0; i < NP; ++i) {
    const int c = (i * 64 + lane) * 8;
    if (c < padded) put(v[i], c);
  }
  for (int c = (NP * 64 + lane) * 8; c < padded; c += 512) {
    Pack8<T> t;
    t.load(xr + c);
    put(t, c);
  }
}

// y[i, h, :] = o[i, h, :] / rms(o[i, h, :]) * w * sigmoid(gate[i, h, :]).  A row of 16 lanes per (token, head); eight
// channels per lane at a time, the first 128 kept in registers.
template <typename T>
__global__ __launch_bounds__(256) void gated_head_norm_kernel(const float* __restrict__ o, const T* __restrict__ gate,
                                                              int64_t ldg, int64_t rows, int heads, int vdim,
                                                              int padded, const float* __restrict__ w, float eps,
                                                              T* __restrict__ y) {
  const int64_t r = (int64_t)blockIdx.x * 16 + (threadIdx.x >> 4);
  const int sub = threadIdx.x & 15;
  const bool ok = r < rows * heads;  // whole rows of lanes: the sum below stays inside one
  const int64_t row = ok ? r / heads : 0, head = ok ? r % heads : 0;
  const float* src = o + (ok ? r : 0) * padded;
  Pack8<float> v;
  v.zero();
  if (sub * 8 < padded) v.load(src + sub * 8);
  float ss = 0.f;
#pragma unroll
  for (int e = 0; e < 8; ++e) ss = __builtin_fmaf(v.get(e), v.get(e), ss);
  for (int c = 128 + sub * 8; c < padded; c += 128) {
    Pack8<float> t;
    t.load(src + c);
#pragma unroll
    for (int e = 0; e < 8; ++e) ss = __builtin_fmaf(t.get(e), t.get(e), ss);
  }
  const float s = 1.f / sqrtf(row16_sum(ss) / vdim + eps);
  if (!ok) return;
  for (int c = sub * 8; c < padded; c += 128) {
    Pack8<float> t = v;
    if (c >= 128) t.load(src + c);
    Pack8<T> g;
    g.load(gate + row * ldg + head * padded + c);
    __attribute__((aligned(16))) T out[8];
#pragma unroll
    for (int e = 0; e < 8; ++e) out[e] = from_f<T>(t.get(e) * s * w[c + e] * sigmoid_f(g.get(e)));
    *reinterpret_cast<Pack8<T>*>(y + r * padded + c) = *reinterpret_cast<const Pack8<T>*>(out);
  }
}

// First index of the largest of `vocab` fp32 logits, and the bookkeeping of a generation loop (one workgroup):
// token <- argmax, sequences[out_index++] <- token, position++, seq_pos++, scores[score_index++] <- logits.
__global__ __launch_bounds__(1024) void greedy_advance_f32_kernel(
    const float* __restrict__ logits, int vocab, int64_t* __restrict__ token, int64_t* __restrict__ position,
    int* __restrict__ seq_pos, int64_t* __restrict__ sequences, int64_t* __restrict__ out_index,
    float* __restrict__ scores, int64_t score_ld, int64_t* __restrict__ score_index, int64_t seq_capacity,
    int64_t score_rows) {
  __shared__ float s_v[16];
  __shared__ int s_i[16];
  float best = -INFINITY;
  int at = 0x7fffffff;
  const int64_t srow = scores ? *score_index : 0;
  const bool keep = scores && srow >= 0 && srow < score_rows;
  for (int i = threadIdx.x; i < vocab; i += blockDim.x) {
    const float v = logits[i];
    if (v > best || at == 0x7fffffff) {
      best = v;
      at = i;
    }
    if (keep) scores[srow * score_ld + i] = v;
  }
  auto merge = [&](float ov, int oi) {
    if (ov > best || (ov == best && oi < at)) {
      best = ov;
      at = oi;
    }
  };
#pragma unroll
  for (int off = 32; off >= 1; off >>= 1) {
    const float ov = __shfl_xor(best, off, kWave);
    const int oi = __shfl_xor(at, off, kWave);
    merge(ov, oi);
  }
  if ((threadIdx.x & 63) == 0) {
    s_v[threadIdx.x >> 6] = best;
    s_i[threadIdx.x >> 6] = at;
  }
  __syncthreads();
  if (threadIdx.x == 0) {
    for (int w = 1; w < (int)(blockDim.x >> 6); ++w) merge(s_v[w], s_i[w]);
    if (at >= vocab) at = 0;
    token[0] = at;
    position[0] += 1;
    seq_pos[0] += 1;
    const int64_t o = out_index[0];
    if (o >= 0 && o < seq_capacity) sequences[o] = at;
    out_index[0] = o + 1;
    if (scores) score_index[0] = srow + 1;
  }
}

}  // namespace dv
