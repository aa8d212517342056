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
  const float c = exp_f(m - mm);
  float den = l * c;
  if (a.sink) den += exp_f(a.sink[head] - mm);
  float f = 1.f / den;
  if (a.gate) f *= sigmoid_f(to_f(reinterpret_cast<const TQ*>(a.gate)[(int64_t)row * a.ldg + head]));
  *rescale = c;
  return f;
}

constexpr int kAttnKeys = 64;

// Grid: (splits, G * chunks of RH query heads, n).
// Keys and values of a tile of 64 are requested together, before the queries are staged, so a split of one tile waits
// for memory once.  With fresh_k / fresh_v this token's key and value come from LDS (and are stored in their slots).
template <typename T, typename TQ, int RH>
__global__ __launch_bounds__(256) void attn_rows_kernel(AttnArgs a) {
  extern __shared__ __attribute__((aligned(16))) unsigned char smem_raw[];
  float* qs = reinterpret_cast<float*>(smem_raw);  // [RH][dim_s]
  float* red = qs + RH * a.dim_s;                  // [256][8]
  T* kf = reinterpret_cast<T*>(red + 256 * 8);     // this token's key [dim_s] and value [vdim_s]
  T* vf = kf + a.dim_s;
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
  const int fresh = a.fresh_k ? pos : -1;
  const T* K = reinterpret_cast<const T*>(a.k) + (int64_t)g * a.k_head;
  const T* V = reinterpret_cast<const T*>(a.v) + (int64_t)g * a.v_head;
  auto slot = [&](int j) -> int64_t { return a.ring > 0 ? j % a.ring : j - a.base; };
  const int nc = a.vdim_s / 8, groups = 256 / nc;
  const int chunk = tid % nc, grp = tid / nc;

  constexpr int VU = 4;  // values a thread keeps of a tile (all of them with at least 16 key groups)
  Pack8<T> kv[4], vv[VU];
  auto load_tile = [&](int jt) {
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      const int j = jt + u * 16 + (tid >> 4);
      if (sub * 8 < a.dim_s && j < j1 && j != fresh) kv[u].load(K + slot(j) * a.ldk + sub * 8);
      else kv[u].zero();
    }
#pragma unroll
    for (int u = 0; u < VU; ++u) {
      const int j = jt + grp + u * groups;
      if (grp < groups && grp + u * groups < kAttnKeys && j < j1 && j != fresh) vv[u].load(V + slot(j) * a.ldv + chunk * 8);
      else vv[u].zero();
    }
  };
  if (j0 < j1) load_tile(j0);

  for (int r = wave; r < RH; r += 4) {
    const TQ* q = reinterpret_cast<const TQ*>(a.q) + (int64_t)row * a.ldq + (int64_t)(h0 + (r < nh ? r : 0)) * a.dim_s;
    float ss = 0.f;
    for (int c = lane; c < a.dim_s; c += 64) {
      const float x = r < nh ? to_f(q[c]) : 0.f;
      qs[r * a.dim_s + c] = x;
      if (c < a.norm_dim) ss = __builtin_fmaf(x, x, ss);
    }
    if (a.norm_dim > 0) {  // a lane reads back what it wrote
      const float s = 1.f / sqrtf(wave_sum(ss) / a.norm_dim + a.eps);
      for (int c = lane; c < a.dim_s; c += 64) qs[r * a.dim_s + c] *= s;
    }
  }
  if (tid < RH) {
    ms[tid] = -1e30f;
    ls[tid] = 0.f;
  }
  if (a.fresh_k && j0 <= pos && pos < j1) {
    const bool first = h0 == g * rep;  // one of the workgroups of a key/value head stores the rows
    if (wave == 2) {
      const float* x = a.fresh_k + (int64_t)g * a.dim_s;
      const float s = a.norm_dim > 0 ? rms_factor(x, a.norm_dim, a.eps, lane) : 1.f;
      T* o = const_cast<T*>(K) + slot(pos) * a.ldk;
      for (int c = lane; c < a.dim_s; c += 64) {
        const T t = from_f<T>(x[c] * s);
        kf[c] = t;
        if (first) o[c] = t;
      }
    } else if (wave == 3) {
      const float* x = a.fresh_v + (int64_t)g * a.vdim_s;
      T* o = const_cast<T*>(V) + slot(pos) * a.ldv;
      for (int c = lane; c < a.vdim_s; c += 64) {
        const T t = from_f<T>(x[c]);
        vf[c] = t;
        if (first) o[c] = t;
      }
    }
  }
  __syncthreads();

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
      Pack8<T> kt[4];
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        const int j = jt + u * 16 + (tid >> 4);
        if (j == fresh && j < j1) kt[u] = *reinterpret_cast<const Pack8<T>*>(kf + c);
        else if (c < 128) kt[u] = kv[u];
        else if (j < j1) kt[u].load(K + slot(j) * a.ldk + c);
        else kt[u].zero();
      }
#pragma unroll
      for (int r = 0; r < RH; ++r) {
        const float4_t qa = *reinterpret_cast<const float4_t*>(qs + r * a.dim_s + c);
        const float4_t qb = *reinterpret_cast<const float4_t*>(qs + r * a.dim_s + c + 4);
#pragma unroll
        for (int u = 0; u < 4; ++u) {
#pragma unroll
          for (int e = 0; e < 4; ++e) s[u][r] = __builtin_fmaf(qa[e], kt[u].get(e), s[u][r]);
#pragma unroll
          for (int e = 0; e < 4; ++e) s[u][r] = __builtin_fmaf(qb[e], kt[u].get(4 + e), s[u][r]);
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
      const float p = in ? exp_f(sc - m1) : 0.f;
      const float sum = wave_sum(p), c = exp_f(m0 - m1);
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
      auto add = [&](const Pack8<T>& x, int i) {
#pragma unroll
        for (int r = 0; r < RH; ++r) {
          const float p = ps[r][i];
#pragma unroll
          for (int e = 0; e < 8; ++e) acc[r][e] = __builtin_fmaf(p, x.get(e), acc[r][e]);
        }
      };
#pragma unroll
      for (int u = 0; u < VU; ++u) {
        const int i = grp + u * groups;
        if (i < cnt) {
          if (jt + i == fresh) add(*reinterpret_cast<const Pack8<T>*>(vf + chunk * 8), i);
          else add(vv[u], i);
        }
      }
      for (int i = grp + VU * groups; i < cnt; i += groups) {
        Pack8<T> x;
        if (jt + i == fresh) x = *reinterpret_cast<const Pack8<T>*>(vf + chunk * 8);
        else x.load(V + slot(jt + i) * a.ldv + chunk * 8);
        add(x, i);
      }
    }
    if (jt + kAttnKeys < j1) load_tile(jt + kAttnKeys);
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

// Adds up the splits of a (row, head): out[row][head][d].  Grid (H, ceil(vdim_s / 64), n); four groups of threads
// share the splits of 64 entries.
constexpr int kMaxSplits = 128;
template <typename TO, typename TQ>
__global__ __launch_bounds__(256) void attn_merge_kernel(AttnArgs a, TO* __restrict__ out) {
  __shared__ float ws[kMaxSplits], acc[4][64], ml[2];
  const int head = blockIdx.x, row = blockIdx.z, stride = a.vdim_s + 2, lane = threadIdx.x & 63, grp = threadIdx.x >> 6;
  const float* p = a.part + ((int64_t)row * a.H + head) * a.splits * stride;
  if (grp == 0) {
    float m0 = -1e30f, m1 = -1e30f, l = 0.f;
    if (lane < a.splits) m0 = p[(int64_t)lane * stride + a.vdim_s];
    if (lane + 64 < a.splits) m1 = p[(int64_t)(lane + 64) * stride + a.vdim_s];
    const float m = butterfly_max<64>(fmaxf(m0, m1));
    const float w0 = exp_f(m0 - m), w1 = exp_f(m1 - m);
    if (lane < a.splits) {
      ws[lane] = w0;
      l = w0 * p[(int64_t)lane * stride + a.vdim_s + 1];
    }
    if (lane + 64 < a.splits) {
      ws[lane + 64] = w1;
      l = __builtin_fmaf(w1, p[(int64_t)(lane + 64) * stride + a.vdim_s + 1], l);
    }
    l = wave_sum(l);
    if (lane == 0) {
      ml[0] = m;
      ml[1] = l;
    }
  }
  __syncthreads();
  const int d = blockIdx.y * 64 + lane;
  float t = 0.f;
  if (d < a.vdim_s) {
#pragma unroll 4
    for (int s = grp; s < a.splits; s += 4) {
      const float w = ws[s];
      if (w > 0.f) t = __builtin_fmaf(p[(int64_t)s * stride + d], w, t);  // splits without tokens hold no sums
    }
  }
  acc[grp][lane] = t;
  __syncthreads();
  if (grp == 0 && d < a.vdim_s) {
    float c;
    const float f = attn_factor<TQ>(a, row, head, ml[0], ml[1], &c);
    out[((int64_t)row * a.H + head) * a.vdim_s + d] = from_f<TO>(((acc[0][lane] + acc[1][lane]) + (acc[2][lane] + acc[3][lane])) * c * f);
  }
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

// Latent attention, one decode row: out[h] = W_uv[h] lat[h], lat fp32 [H][rank].  Grid (H, row parts).
template <typename T>
__global__ __launch_bounds__(256) void latent_out_kernel(const float* __restrict__ lat_all, const T* __restrict__ W,
                                                         int rank, int vrows, T* __restrict__ out) {
  extern __shared__ __attribute__((aligned(16))) unsigned char smem_raw[];
  float* lat = reinterpret_cast<float*>(smem_raw);
  const int head = blockIdx.x, lane = threadIdx.x & 63;
  for (int d = threadIdx.x; d < rank; d += 256) lat[d] = lat_all[(int64_t)head * rank + d];
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
