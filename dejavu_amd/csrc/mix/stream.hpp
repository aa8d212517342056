// Elementwise kernels around the fp32 residual stream: embedding, dynamic tanh, gated feed-forward activation.
#pragma once
#include "elem.hpp"

namespace dv {

// x = x0 = embed[token]; h = norm(x).  One workgroup per token.
template <typename T>
__global__ __launch_bounds__(256) void embed_norm_kernel(const int64_t* __restrict__ tokens, int64_t vocab,
                                                         const T* __restrict__ embed, int width, float* __restrict__ x,
                                                         float* __restrict__ x0, DynTanh norm, T* __restrict__ h) {
  const int64_t i = blockIdx.x;
  const int64_t tok = tokens[i];
  const bool ok = tok >= 0 && tok < vocab;
  for (int c = threadIdx.x; c < width; c += blockDim.x) {
    const float v = ok ? to_f(embed[tok * width + c]) : 0.f;
    x[i * width + c] = v;
    if (x0) x0[i * width + c] = v;
    h[i * width + c] = from_f<T>(dyn_tanh(v, norm, c));
  }
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

// y == nullptr: only x += x0 and h = pre(x).
template <typename T>
__global__ __launch_bounds__(256) void residual_norm_kernel(const T* __restrict__ y, int64_t count, int width,
                                                            ResidualArgs a) {
  for (int64_t at = (int64_t)blockIdx.x * 256 + threadIdx.x; at < count; at += (int64_t)gridDim.x * 256) {
    const int c = (int)(at % width);
    if (y) {
      residual_apply<T>(a, at, c, to_f(y[at]));
    } else {
      float v = a.x[at];
      if (a.x0) v += a.x0[at];
      a.x[at] = v;
      if (a.h) reinterpret_cast<T*>(a.h)[at] = from_f<T>(dyn_tanh(v, a.pre, c));
    }
  }
}

// Clamped gated unit of one (gate, up) pair.
__device__ __forceinline__ float clamped_glu_f(float g, float u, float limit) {
  g = fminf(g, limit);
  u = fminf(fmaxf(u, -limit), limit);
  return g * sigmoid_f(1.702f * g) * (u + 1.f);
}

// y[i] from gu[2 i] (gate) and gu[2 i + 1] (up); four outputs per thread, count % 4 == 0.
template <typename T>
__global__ __launch_bounds__(256) void clamped_glu_kernel(const T* __restrict__ gu, int64_t count, float limit,
                                                          T* __restrict__ y) {
  const int64_t i = ((int64_t)blockIdx.x * 256 + threadIdx.x) * 4;
  if (i >= count) return;
  Pack8<T> v;
  v.load(gu + 2 * i);
#pragma unroll
  for (int e = 0; e < 4; ++e) y[i + e] = from_f<T>(clamped_glu_f(v.get(2 * e), v.get(2 * e + 1), limit));
}

// y = x * rsqrt(mean(x^2) + eps) * w over the first `dim` entries of every row (entries up to ldy: weight 0).
// One wave per row.
template <typename T>
__global__ __launch_bounds__(256) void rms_rows_kernel(const T* __restrict__ x, int64_t ldx, int64_t rows, int dim,
                                                       int padded, const float* __restrict__ w, float eps,
                                                       T* __restrict__ y, int64_t ldy) {
  const int64_t r = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
  if (r >= rows) return;
  const int lane = threadIdx.x & 63;
  float ss = 0.f;
  for (int c = lane; c < dim; c += 64) {
    const float v = to_f(x[r * ldx + c]);
    ss = __builtin_fmaf(v, v, ss);
  }
  const float s = 1.f / sqrtf(wave_sum(ss) / dim + eps);
  for (int c = lane; c < padded; c += 64) y[r * ldy + c] = from_f<T>(to_f(x[r * ldx + c]) * s * w[c]);
}

// y[i, h, :] = o[i, h, :] / rms(o[i, h, :]) * w * sigmoid(gate[i, h, :]); one wave per (token, head).
template <typename T>
__global__ __launch_bounds__(256) void gated_head_norm_kernel(const float* __restrict__ o, const T* __restrict__ gate,
                                                              int64_t ldg, int64_t rows, int heads, int vdim,
                                                              int padded, const float* __restrict__ w, float eps,
                                                              T* __restrict__ y) {
  const int64_t r = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
  if (r >= rows * heads) return;
  const int lane = threadIdx.x & 63;
  const int64_t row = r / heads, head = r % heads;
  float ss = 0.f;
  for (int c = lane; c < vdim; c += 64) ss = __builtin_fmaf(o[r * padded + c], o[r * padded + c], ss);
  const float s = 1.f / sqrtf(wave_sum(ss) / vdim + eps);
  for (int c = lane; c < padded; c += 64)
    y[r * padded + c] = from_f<T>(o[r * padded + c] * s * w[c] * sigmoid_f(to_f(gate[row * ldg + head * padded + c])));
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
