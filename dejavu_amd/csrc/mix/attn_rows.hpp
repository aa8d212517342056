// Softmax attention of single query rows on the vector ALUs: decode steps (keys in a ring or in a latent cache,
// split over workgroups) and, in fp32, the rows of a prompt.  Arithmetic fp32.
#pragma once
#include "elem.hpp"

namespace dv {

using AttnArgs = dvAttnArgs;

__device__ __forceinline__ float rms_factor(const float* x, int dim, float eps, int lane) {
  float ss = 0.f;
  for (int c = lane; c < dim; c += 64) ss = __builtin_fmaf(x[c], x[c], ss);
  return 1.f / sqrtf(wave_sum(ss) / dim + eps);
}

// Final value of a head: sums / (denominator + exp(sink)), times the gate.
template <typename TQ>
__device__ __forceinline__ float attn_factor(const AttnArgs& a, int row, int head, float m, float l, float* rescale) {
  float mm = m;
  if (a.sink) mm = fmaxf(mm, a.sink[head]);
  const float c = expf(m - mm);
  float den = l * c;
  if (a.sink) den += expf(a.sink[head] - mm);
  float f = 1.f / den;
  if (a.gate) f *= sigmoid_f(to_f(reinterpret_cast<const TQ*>(a.gate)[(int64_t)row * a.ldg + head]));
  *rescale = c;
  return f;
}

constexpr int kAttnKeys = 64;

// Grid: (splits, G * chunks of RH query heads, n).
template <typename T, typename TQ, int RH>
__global__ __launch_bounds__(256) void attn_rows_kernel(AttnArgs a) {
  extern __shared__ __attribute__((aligned(16))) unsigned char smem_raw[];
  float* qs = reinterpret_cast<float*>(smem_raw);  // [RH][dim_s]
  float* red = qs + RH * a.dim_s;                  // [256][8]
  __shared__ float ps[RH][kAttnKeys], corr[RH], ms[RH], ls[RH];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, sub = tid & 15;
  const int rep = a.H / a.G, chunks = (rep + RH - 1) / RH;
  const int g = blockIdx.y / chunks, h0 = g * rep + (blockIdx.y % chunks) * RH;
  const int nh = min(RH, (g + 1) * rep - h0);
  const int row = blockIdx.z, split = blockIdx.x;
  const int pos = seq_position(a.pos_dev, a.pos_host) + row;
  const int lo = a.window > 0 ? max(0, pos - a.window + 1) : 0;
  const int nk = pos + 1 - lo;
  const int per = ((nk + a.splits - 1) / a.splits + kAttnKeys - 1) / kAttnKeys * kAttnKeys;
  const int j0 = lo + split * per, j1 = min(pos + 1, j0 + per);
  const T* K = reinterpret_cast<const T*>(a.k) + (int64_t)g * a.k_head;
  const T* V = reinterpret_cast<const T*>(a.v) + (int64_t)g * a.v_head;
  auto slot = [&](int j) -> int64_t { return a.ring > 0 ? j % a.ring : j - a.base; };

  for (int r = wave; r < RH; r += 4) {
    const TQ* q = reinterpret_cast<const TQ*>(a.q) + (int64_t)row * a.ldq + (int64_t)(h0 + (r < nh ? r : 0)) * a.dim_s;
    for (int c = lane; c < a.dim_s; c += 64) qs[r * a.dim_s + c] = r < nh ? to_f(q[c]) : 0.f;
  }
  if (tid < RH) {
    ms[tid] = -1e30f;
    ls[tid] = 0.f;
  }
  if (a.fresh_k && j0 <= pos && pos < j1) {
    if (wave == 0) {
      const float* x = a.fresh_k + (int64_t)g * a.dim_s;
      const float s = a.norm_dim > 0 ? rms_factor(x, a.norm_dim, a.eps, lane) : 1.f;
      T* o = const_cast<T*>(K) + slot(pos) * a.ldk;
      for (int c = lane; c < a.dim_s; c += 64) o[c] = from_f<T>(x[c] * s);
    } else if (wave == 1) {
      const float* x = a.fresh_v + (int64_t)g * a.vdim_s;
      T* o = const_cast<T*>(V) + slot(pos) * a.ldv;
      for (int c = lane; c < a.vdim_s; c += 64) o[c] = from_f<T>(x[c]);
    }
    __threadfence_block();
  }
  __syncthreads();
  if (a.norm_dim > 0) {
    for (int r = wave; r < nh; r += 4) {
      const float s = rms_factor(qs + r * a.dim_s, a.norm_dim, a.eps, lane);
      for (int c = lane; c < a.dim_s; c += 64) qs[r * a.dim_s + c] *= s;
    }
    __syncthreads();
  }

  const int nc = a.vdim_s / 8, groups = 256 / nc;
  const int chunk = tid % nc, grp = tid / nc;
  float acc[RH][8];
#pragma unroll
  for (int r = 0; r < RH; ++r)
#pragma unroll
    for (int e = 0; e < 8; ++e) acc[r][e] = 0.f;

  for (int jt = j0; jt < j1; jt += kAttnKeys) {
    // scores: a row of 16 lanes per key, four keys each
    float s[4][RH];
#pragma unroll
    for (int u = 0; u < 4; ++u)
#pragma unroll
      for (int r = 0; r < RH; ++r) s[u][r] = 0.f;
    for (int c = sub * 8; c < a.dim_s; c += 128) {
      Pack8<T> kv[4];
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        const int j = jt + u * 16 + (tid >> 4);
        if (j < j1) kv[u].load(K + slot(j) * a.ldk + c);
        else kv[u].zero();
      }
#pragma unroll
      for (int r = 0; r < RH; ++r) {
        const float4_t qa = *reinterpret_cast<const float4_t*>(qs + r * a.dim_s + c);
        const float4_t qb = *reinterpret_cast<const float4_t*>(qs + r * a.dim_s + c + 4);
#pragma unroll
        for (int u = 0; u < 4; ++u) {
#pragma unroll
          for (int e = 0; e < 4; ++e) s[u][r] = __builtin_fmaf(qa[e], kv[u].get(e), s[u][r]);
#pragma unroll
          for (int e = 0; e < 4; ++e) s[u][r] = __builtin_fmaf(qb[e], kv[u].get(4 + e), s[u][r]);
        }
      }
    }
#pragma unroll
    for (int u = 0; u < 4; ++u)
#pragma unroll
      for (int r = 0; r < RH; ++r) {
        const float d = row16_sum(s[u][r]);
        if (sub == (r & 15)) ps[r][u * 16 + (tid >> 4)] = d * a.scale;
      }
    __syncthreads();
    for (int r = wave; r < RH; r += 4) {
      const bool in = jt + lane < j1;
      const float sc = in ? ps[r][lane] : -INFINITY;
      const float m0 = ms[r], m1 = fmaxf(m0, butterfly_max<64>(sc));
      const float p = in ? expf(sc - m1) : 0.f;
      const float sum = wave_sum(p), c = expf(m0 - m1);
      ps[r][lane] = p;
      if (lane == 0) {
        ms[r] = m1;
        ls[r] = ls[r] * c + sum;
        corr[r] = c;
      }
    }
    __syncthreads();
    if (grp < groups) {
#pragma unroll
      for (int r = 0; r < RH; ++r) {
        const float c = corr[r];
#pragma unroll
        for (int e = 0; e < 8; ++e) acc[r][e] *= c;
      }
      const int cnt = min(kAttnKeys, j1 - jt);
#pragma unroll 4
      for (int i = grp; i < cnt; i += groups) {
        Pack8<T> vv;
        vv.load(V + slot(jt + i) * a.ldv + chunk * 8);
#pragma unroll
        for (int r = 0; r < RH; ++r) {
          const float p = ps[r][i];
#pragma unroll
          for (int e = 0; e < 8; ++e) acc[r][e] = __builtin_fmaf(p, vv.get(e), acc[r][e]);
        }
      }
    }
    __syncthreads();
  }
  // the key groups of a head are added up in LDS, one head at a time
#pragma unroll
  for (int r = 0; r < RH; ++r) {
    if (r < nh) {
#pragma unroll
      for (int e = 0; e < 8; ++e) red[tid * 8 + e] = acc[r][e];
      __syncthreads();
      const int head = h0 + r;
      float c = 1.f, f = 1.f;
      if (a.splits == 1) f = attn_factor<TQ>(a, row, head, ms[r], ls[r], &c);
      for (int d = tid; d < a.vdim_s; d += 256) {
        float t = 0.f;
        for (int i = 0; i < groups; ++i) t += red[(i * nc + d / 8) * 8 + (d & 7)];
        if (a.splits == 1) {
          reinterpret_cast<T*>(a.out)[((int64_t)row * a.H + head) * a.vdim_s + d] = from_f<T>(t * c * f);
        } else {
          a.part[(((int64_t)row * a.H + head) * a.splits + split) * (a.vdim_s + 2) + d] = t;
        }
      }
      if (a.splits > 1 && tid == 0) {
        float* p = a.part + (((int64_t)row * a.H + head) * a.splits + split) * (a.vdim_s + 2) + a.vdim_s;
        p[0] = ms[r];
        p[1] = ls[r];
      }
      __syncthreads();
    }
  }
}

// Adds up the splits of one (row, head): sums[d] over LDS-free reads; returns through `val` for entry d.
struct SplitMerge {
  float m, l;
};
__device__ __forceinline__ SplitMerge merge_splits(const float* __restrict__ p, int splits, int stride, int vdim_s) {
  SplitMerge r{-1e30f, 0.f};
  for (int s = 0; s < splits; ++s) r.m = fmaxf(r.m, p[(int64_t)s * stride + vdim_s]);
  for (int s = 0; s < splits; ++s)
    r.l += p[(int64_t)s * stride + vdim_s + 1] * expf(p[(int64_t)s * stride + vdim_s] - r.m);
  return r;
}
__device__ __forceinline__ float merged_value(const float* __restrict__ p, int splits, int stride, int vdim_s, int d,
                                              float m) {
  float t = 0.f;
  for (int s = 0; s < splits; ++s) t += p[(int64_t)s * stride + d] * expf(p[(int64_t)s * stride + vdim_s] - m);
  return t;
}

// One workgroup per (head, row).
template <typename T, typename TQ>
__global__ __launch_bounds__(256) void attn_merge_kernel(AttnArgs a) {
  const int head = blockIdx.x, row = blockIdx.y, stride = a.vdim_s + 2;
  const float* p = a.part + ((int64_t)row * a.H + head) * a.splits * stride;
  const SplitMerge sm = merge_splits(p, a.splits, stride, a.vdim_s);
  float c;
  const float f = attn_factor<TQ>(a, row, head, sm.m, sm.l, &c);
  for (int d = threadIdx.x; d < a.vdim_s; d += 256)
    reinterpret_cast<T*>(a.out)[((int64_t)row * a.H + head) * a.vdim_s + d] =
        from_f<T>(merged_value(p, a.splits, stride, a.vdim_s, d, sm.m) * c * f);
}

// Latent attention, one decode row: the query of head h in the latent space, sum_d W_uk[h, d, :] q[h, d].
// Grid (H, ceil(rank / 128)).
template <typename T>
__global__ __launch_bounds__(256) void latent_absorb_kernel(const float* __restrict__ q, const T* __restrict__ W,
                                                            int dim_s, int rank, float* __restrict__ out) {
  __shared__ float red[16][128];
  const int head = blockIdx.x, c = (threadIdx.x & 15) * 8, grp = threadIdx.x >> 4;
  const int col = blockIdx.y * 128 + c;
  float acc[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
  if (col < rank) {
#pragma unroll 4
    for (int d = grp; d < dim_s; d += 16) {
      Pack8<T> w;
      w.load(W + ((int64_t)head * dim_s + d) * rank + col);
      const float qv = q[head * dim_s + d];
#pragma unroll
      for (int e = 0; e < 8; ++e) acc[e] = __builtin_fmaf(w.get(e), qv, acc[e]);
    }
  }
#pragma unroll
  for (int e = 0; e < 8; ++e) red[grp][c + e] = acc[e];
  __syncthreads();
  for (int i = threadIdx.x; i < 128; i += 256) {
    if (blockIdx.y * 128 + i < rank) {
      float t = 0.f;
#pragma unroll
      for (int k = 0; k < 16; ++k) t += red[k][i];
      out[(int64_t)head * rank + blockIdx.y * 128 + i] = t;
    }
  }
}

// Latent attention, one decode row: merges the splits of head h and applies W_uv[h] and the gate.
// a.vdim_s is the latent's size here; grid (H, row parts).
template <typename T>
__global__ __launch_bounds__(256) void latent_out_kernel(AttnArgs a, const T* __restrict__ W, int vrows, T* out) {
  extern __shared__ __attribute__((aligned(16))) unsigned char smem_raw[];
  float* lat = reinterpret_cast<float*>(smem_raw);
  const int head = blockIdx.x, rank = a.vdim_s, stride = rank + 2, lane = threadIdx.x & 63;
  const float* p = a.part + (int64_t)head * a.splits * stride;
  const SplitMerge sm = merge_splits(p, a.splits, stride, rank);
  float c;
  const float f = attn_factor<float>(a, 0, head, sm.m, sm.l, &c) * c;
  for (int d = threadIdx.x; d < rank; d += 256) lat[d] = merged_value(p, a.splits, stride, rank, d, sm.m) * f;
  __syncthreads();
  for (int r = blockIdx.y * 4 + (threadIdx.x >> 6); r < vrows; r += gridDim.y * 4) {
    const T* w = W + ((int64_t)head * vrows + r) * rank;
    float acc = 0.f;
    for (int i = lane * 8; i < rank; i += 512) {
      Pack8<T> v;
      v.load(w + i);
#pragma unroll
      for (int e = 0; e < 8; ++e) acc = __builtin_fmaf(v.get(e), lat[i + e], acc);
    }
    acc = wave_sum(acc);
    if (lane == 0) out[(int64_t)head * vrows + r] = from_f<T>(acc);
  }
}

// Copies rows of keys or values between a portion's buffer and a ring: dst row of token j is slot(j).
//   to_ring : ring[(first + i) % cap] <- buf[at + i]       from ring: buf[at + i] <- ring[(first + i) % cap]
template <typename T>
__global__ __launch_bounds__(256) void ring_copy_kernel(T* __restrict__ buf, int64_t ldb, T* __restrict__ ring, int cap,
                                                        int64_t ldr, int first, int count, int width, int to_ring) {
  const int vecs = width / 8;
  const int64_t total = (int64_t)count * vecs;
  for (int64_t at = (int64_t)blockIdx.x * 256 + threadIdx.x; at < total; at += (int64_t)gridDim.x * 256) {
    const int i = (int)(at / vecs), c = (int)(at % vecs) * 8;
    T* b = buf + (int64_t)i * ldb + c;
    T* r = ring + (int64_t)((first + i) % cap) * ldr + c;
    if (to_ring) *reinterpret_cast<Pack8<T>*>(r) = *reinterpret_cast<const Pack8<T>*>(b);
    else *reinterpret_cast<Pack8<T>*>(b) = *reinterpret_cast<const Pack8<T>*>(r);
  }
}

}  // namespace dv
