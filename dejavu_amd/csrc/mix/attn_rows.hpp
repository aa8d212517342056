// Softmax attention of single query rows on the vector ALUs: decode steps (keys in a ring or in a latent cache,
// split over workgroups) and, in fp32, the rows of a prompt.  Arithmetic fp32.
#pragma once
#include "elem.hpp"

namespace dv {

using AttnArgs = dvAttnArgs;

// The oldest position that the query at `pos` sees.
__device__ __forceinline__ int oldest_key(const AttnArgs& a, int pos) {
  if (a.window > 0) return max(0, pos - a.window + 1);
  return a.chunk > 0 ? pos - pos % a.chunk : 0;
}

// By one wave: put(c, x[c] / rms(x) * w[c]) for every entry, the mean over norm_dim entries (0: put(c, x[c])); w may be
// null.
template <typename T, typename F>
__device__ __forceinline__ void normed_row(const T* __restrict__ x, int n, int norm_dim, float eps,
                                           const float* __restrict__ w, int lane, F put) {
  constexpr int NX = 4;  // values a lane keeps; longer rows read the rest again
  float v[NX], wv[NX];
#pragma unroll
  for (int u = 0; u < NX; ++u) {
    v[u] = to_f(x[min(lane + u * 64, n - 1)]);
    wv[u] = w ? w[min(lane + u * 64, n - 1)] : 1.f;
  }
  float s = 1.f;
  if (norm_dim > 0) {
    float ss = 0.f;
#pragma unroll
    for (int u = 0; u < NX; ++u)
      if (lane + u * 64 < norm_dim) ss = __builtin_fmaf(v[u], v[u], ss);
    for (int c = lane + NX * 64; c < norm_dim; c += 64) ss = __builtin_fmaf(to_f(x[c]), to_f(x[c]), ss);
    s = 1.f / sqrtf(wave_sum(ss) / norm_dim + eps);
  }
#pragma unroll
  for (int u = 0; u < NX; ++u)
    if (lane + u * 64 < n) put(lane + u * 64, v[u] * s * wv[u]);
  for (int c = lane + NX * 64; c < n; c += 64) put(c, to_f(x[c]) * s * (w ? w[c] : 1.f));
}

// Partial sums of a split: `part` holds [n][H][splits][vdim_s] sums, then [n][H][splits][2] (maximum, denominator).
__device__ __forceinline__ float* part_sums(const AttnArgs& a, int row, int head, int split) {
  return a.part + (((int64_t)row * a.H + head) * a.splits + split) * a.vdim_s;
}
__device__ __forceinline__ float* part_ml(const AttnArgs& a, int row, int head, int split) {
  return a.part + (int64_t)a.n * a.H * a.splits * a.vdim_s + (((int64_t)row * a.H + head) * a.splits + split) * 2;
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

// Floats for the sums of the key groups at the end of attn_rows_kernel.
__host__ __device__ inline int attn_red_floats(int rh, int vdim_s) {
  return vdim_s <= 256 && 4 * rh * vdim_s > 256 * 8 ? 4 * rh * vdim_s : 256 * 8;
}

// Grid: (splits, G * chunks of RH query heads, n).
// Keys and values of a tile of 64 are requested together, before the queries are staged, so a split of one tile waits
// for memory once.  With fresh_k / fresh_v this token's key and value come from LDS (and are stored in their slots).
template <typename T, typename TQ, int RH>
__global__ __launch_bounds__(256) void attn_rows_kernel(AttnArgs a) {
  extern __shared__ __attribute__((aligned(16))) unsigned char smem_raw[];
  float* qs = reinterpret_cast<float*>(smem_raw);  // [RH][dim_s]
  float* red = qs + RH * a.dim_s;
  T* kf = reinterpret_cast<T*>(red + attn_red_floats(RH, a.vdim_s));     // this token's key [dim_s] and value [vdim_s]
  T* vf = kf + a.dim_s;
  __shared__ float ps[RH][kAttnKeys], corr[RH], ms[RH], ls[RH];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, sub = tid & 15;
  const int rep = a.H / a.G, chunks = (rep + RH - 1) / RH;
  const int g = blockIdx.y / chunks, h0 = g * rep + (blockIdx.y % chunks) * RH;
  const int nh = min(RH, (g + 1) * rep - h0);
  const int row = blockIdx.z, split = blockIdx.x;
  const int pos = seq_position(a.pos_dev, a.pos_host) + row;
  const int lo = oldest_key(a, pos);
  const int nk = pos + 1 - lo;
  const int per = ((nk + a.splits - 1) / a.splits + kAttnKeys - 1) / kAttnKeys * kAttnKeys;
  const int j0 = lo + split * per, j1 = min(pos + 1, j0 + per);
  const int fresh = a.fresh_k ? pos : -1;
  const T* K = reinterpret_cast<const T*>(a.k) + (int64_t)g * a.k_head;
  const T* V = reinterpret_cast<const T*>(a.v) + (int64_t)g * a.v_head;
  // keys of a split lie in consecutive slots but for one wrap (a ring holds at least the window or chunk)
  const int s0 = a.ring > 0 ? j0 % a.ring : j0 - a.base;
  auto slot = [&](int j) -> int64_t {
    const int s = s0 + (j - j0);
    return a.ring > 0 && s >= a.ring ? s - a.ring : s;
  };
  const int nc = a.vdim_s / 8;
  const bool pow2 = nc <= 32 && (nc & (nc - 1)) == 0;
  const int sh = 31 - __builtin_clz(nc);
  const int groups = pow2 ? 256 >> sh : 256 / nc;
  const int grp = pow2 ? tid >> sh : tid / nc, chunk = pow2 ? tid & (nc - 1) : tid - grp * nc;

  constexpr int VU = 4;  // values a thread keeps of a tile (all of them with at least 16 key groups)
  constexpr int RW = (RH + 3) / 4;  // heads whose softmax a wave does
  Pack8<T> kv[4], vv[VU];
  float rb[RW];  // their biases for key `lane` of a tile
  auto load_tile = [&](int jt) {
#pragma unroll
    for (int u = 0; u < RW; ++u) {
      rb[u] = 0.f;
      if (a.rel) {
        const int r = min(wave + u * 4, nh - 1), n = min(max(pos - jt - lane, 0), a.rel_len - 1);
        rb[u] = a.rel[(int64_t)(h0 + r) * a.rel_len + n];
      }
    }
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      const int j = min(jt + u * 16 + (tid >> 4), j1 - 1);
      kv[u].load(K + slot(j) * a.ldk + min(sub * 8, a.dim_s - 8));
    }
#pragma unroll
    for (int u = 0; u < VU; ++u) {
      const int j = min(jt + grp + u * groups, j1 - 1);
      vv[u].load(V + slot(j) * a.ldv + chunk * 8);
    }
  };
  if (j0 < j1) load_tile(j0);

  for (int r = wave; r < RH; r += 4) {
    const TQ* q = reinterpret_cast<const TQ*>(a.q) + (int64_t)row * a.ldq + (int64_t)(h0 + (r < nh ? r : 0)) * a.dim_s;
    const bool normed = a.norm_dim > 0;
    normed_row(q, a.dim_s, normed ? a.norm_dim : 0, a.eps, a.q_w, lane,
               [&](int c, float x) { qs[r * a.dim_s + c] = r < nh ? x : 0.f; });
  }
  if (tid < RH) {
    ms[tid] = -1e30f;
    ls[tid] = 0.f;
  }
  if (a.fresh_k && j0 <= pos && pos < j1) {
    const bool first = h0 == g * rep;  // one of the workgroups of a key/value head stores the rows
    if (wave == 2) {
      T* o = const_cast<T*>(K) + slot(pos) * a.ldk;
      normed_row(a.fresh_k + (int64_t)g * a.dim_s, a.dim_s, a.norm_dim, a.eps, a.k_w, lane, [&](int c, float x) {
        const T t = from_f<T>(x);
        kf[c] = t;
        if (first) o[c] = t;
      });
    } else if (wave == 3) {
      T* o = const_cast<T*>(V) + slot(pos) * a.ldv;
      const float* other = a.other_v ? a.other_v + (int64_t)g * a.vdim_s : nullptr;
      const float lam = other ? *a.lambda : 0.f;
      normed_row(a.fresh_v + (int64_t)g * a.vdim_s, a.vdim_s, 0, 0.f, nullptr, lane, [&](int c, float x) {
        if (other) x = __builtin_fmaf(lam, other[c], (1.f - lam) * x);
        const T t = from_f<T>(x);
        vf[c] = t;
        if (first) o[c] = t;
      });
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
        else kt[u].load(K + slot(min(j, j1 - 1)) * a.ldk + c);
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
#pragma unroll
    for (int u = 0; u < RW; ++u) {
      const int r = wave + u * 4;
      if (r >= RH) break;
      const bool in = jt + lane < j1;
      const float sc = in ? ps[r][lane] + rb[u] : -INFINITY;
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
  // The key groups are added up: inside a wave by exchanges where whole groups lie side by side in it, the rest in
  // LDS, a head at a time.
  if (pow2) {
    for (int off = 32; off >= nc; off >>= 1) {
#pragma unroll
      for (int r = 0; r < RH; ++r)
#pragma unroll
        for (int e = 0; e < 8; ++e) acc[r][e] += __shfl_xor(acc[r][e], off, kWave);
    }
  }
  auto finish = [&](int r, int d, float t) {
    const int head = h0 + r;
    if (a.splits == 1) {
      float c;
      const float f = attn_factor<TQ>(a, row, head, ms[r], ls[r], &c);
      reinterpret_cast<T*>(a.out)[((int64_t)row * a.H + head) * a.vdim_s + d] = from_f<T>(t * c * f);
    } else {
      part_sums(a, row, head, split)[d] = t;
      if (d == 0) {
        float* p = part_ml(a, row, head, split);
        p[0] = ms[r];
        p[1] = ls[r];
      }
    }
  };
  if (pow2) {
    // red holds [4 waves][RH][vdim_s] (at most 4 * RH * 256 floats)
    if (lane < nc) {
#pragma unroll
      for (int r = 0; r < RH; ++r)
#pragma unroll
        for (int e = 0; e < 8; ++e) red[(wave * RH + r) * a.vdim_s + lane * 8 + e] = acc[r][e];
    }
    __syncthreads();
    for (int i = tid; i < nh * a.vdim_s; i += 256) {
      const int r = i >> (sh + 3), d = i & (a.vdim_s - 1);
      float t = 0.f;
      for (int w = 0; w < 4; ++w) t += red[(w * RH + r) * a.vdim_s + d];
      finish(r, d, t);
    }
    return;
  }
#pragma unroll
  for (int r = 0; r < RH; ++r) {
    if (r < nh) {
#pragma unroll
      for (int e = 0; e < 8; ++e) red[tid * 8 + e] = acc[r][e];
      __syncthreads();
      for (int d = tid; d < a.vdim_s; d += 256) {
        float t = 0.f;
        for (int i = 0; i < groups; ++i) t += red[(i * nc + d / 8) * 8 + (d & 7)];
        finish(r, d, t);
      }
      __syncthreads();
    }
  }
}

// Adds up the splits of a (row, head): out[row][head][d].  Grid (H, ceil(vdim_s / 64), n); four groups of threads
// share the splits of 64 entries.
constexpr int kMaxSplits = 128;
// By one wave: the weight of every split, and the maximum and denominator of all.
__device__ __forceinline__ void split_weights(const float* __restrict__ p, int splits, int lane, float* ws, float* ml) {
  const bool in0 = lane < splits, in1 = lane + 64 < splits;
  const float* p0 = p + (in0 ? lane : 0) * 2;
  const float* p1 = p + (in1 ? lane + 64 : 0) * 2;
  const float a0 = p0[0], b0 = p0[1], a1 = p1[0], b1 = p1[1];
  const float m0 = in0 ? a0 : -1e30f, l0 = in0 ? b0 : 0.f, m1 = in1 ? a1 : -1e30f, l1 = in1 ? b1 : 0.f;
  const float m = butterfly_max<64>(fmaxf(m0, m1));
  const float w0 = exp_f(m0 - m), w1 = exp_f(m1 - m);
  if (in0) ws[lane] = w0;
  if (in1) ws[lane + 64] = w1;
  const float l = wave_sum(w0 * l0 + w1 * l1);
  if (lane == 0) {
    ml[0] = m;
    ml[1] = l;
  }
}
template <typename TO, typename TQ>
__global__ __launch_bounds__(256) void attn_merge_kernel(AttnArgs a, TO* __restrict__ out) {
  __shared__ float ws[kMaxSplits], acc[4][64], ml[2];
  const int head = blockIdx.x, row = blockIdx.z, stride = a.vdim_s, lane = threadIdx.x & 63, grp = threadIdx.x >> 6;
  const float* p = part_sums(a, row, head, 0);
  const int d = blockIdx.y * 64 + lane;
  constexpr int PV = 16;  // sums requested before the weights are known
  float v[PV];
#pragma unroll
  for (int i = 0; i < PV; ++i) v[i] = p[(int64_t)min(grp + 4 * i, a.splits - 1) * stride + min(d, a.vdim_s - 1)];
  if (grp == 0) split_weights(part_ml(a, row, head, 0), a.splits, lane, ws, ml);
  __syncthreads();
  float t = 0.f;
#pragma unroll
  for (int i = 0; i < PV; ++i)
    if (grp + 4 * i < a.splits) t = __builtin_fmaf(v[i], ws[grp + 4 * i], t);
  if (d < a.vdim_s)
    for (int s = grp + 4 * PV; s < a.splits; s += 4) t = __builtin_fmaf(p[(int64_t)s * stride + d], ws[s], t);
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

// Latent attention, one decode row: merges the splits of head h, gates, and applies W_uv[h].  Grid (H, row parts):
// every part merges the whole latent for itself.  The first weights are requested before anything else.
template <typename T>
__global__ __launch_bounds__(256) void latent_out_kernel(AttnArgs a, const T* __restrict__ W, int vrows, T* __restrict__ out) {
  extern __shared__ __attribute__((aligned(16))) unsigned char smem_raw[];
  float* sums = reinterpret_cast<float*>(smem_raw);  // [thread groups][rank]
  __shared__ float ws[kMaxSplits], ml[2];
  const int head = blockIdx.x, rank = a.vdim_s, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const float* p = part_sums(a, 0, head, 0);
  constexpr int PR = 8;  // weight rows a wave takes at a time
  Pack8<T> w[PR];
  const int r0 = blockIdx.y * 4 + wave, rstep = gridDim.y * 4;
  const T* wh = W + (int64_t)head * vrows * rank;
  auto load_rows = [&](int r) {
#pragma unroll
    for (int i = 0; i < PR; ++i) w[i].load(wh + min(r + i * rstep, vrows - 1) * rank + min(lane * 8, rank - 8));
  };
  load_rows(r0);
  // four channels per thread; the thread groups share the splits, eight of them requested together
  const int nv = rank / 4, ng = nv < 256 ? 256 / nv : 1, grp = threadIdx.x / nv, v0 = threadIdx.x % nv;
  const bool batch = a.splits >= 8 * ng && grp < ng;  // the first eight before the weights are known
  float4_t first[8];
  if (batch) {
#pragma unroll
    for (int u = 0; u < 8; ++u) first[u] = *reinterpret_cast<const float4_t*>(p + (grp + u * ng) * rank + v0 * 4);
  }
  if (wave == 0) split_weights(part_ml(a, 0, head, 0), a.splits, lane, ws, ml);
  __syncthreads();
  float c;
  const float f = attn_factor<float>(a, 0, head, ml[0], ml[1], &c) * c;
  const int step = ng * rank;
  for (int v = v0; v < nv; v += 256) {  // one turn unless the latent has more than 1024 channels
    if (grp < ng) {
      float4_t t = {0.f, 0.f, 0.f, 0.f};
      const float* q = p + grp * rank + v * 4;
      int s = grp;
      if (batch && v == v0) {
#pragma unroll
        for (int u = 0; u < 8; ++u) t += first[u] * ws[s + u * ng];
        s += 8 * ng;
        q += 8 * step;
      }
      for (; s + 7 * ng < a.splits; s += 8 * ng, q += 8 * step) {
        float4_t x[8];
#pragma unroll
        for (int u = 0; u < 8; ++u) x[u] = *reinterpret_cast<const float4_t*>(q + u * step);
#pragma unroll
        for (int u = 0; u < 8; ++u) t += x[u] * ws[s + u * ng];
      }
      for (; s < a.splits; s += ng, q += step) t += *reinterpret_cast<const float4_t*>(q) * ws[s];
      *reinterpret_cast<float4_t*>(sums + (grp * nv + v) * 4) = t * f;
    }
  }
  __syncthreads();
  if (ng > 1) {
    for (int d = threadIdx.x; d < rank; d += 256) {
      float t = sums[d];
      for (int g = 1; g < ng; ++g) t += sums[g * rank + d];
      sums[d] = t;  // only this thread reads entry d of the other groups
    }
    __syncthreads();
  }
  const float* lat = sums;
  for (int r = r0; r < vrows; r += PR * rstep) {
    float sum[PR];
#pragma unroll
    for (int i = 0; i < PR; ++i) sum[i] = 0.f;
    if (lane * 8 < rank) {
      Pack8<float> x;
      x.load(lat + lane * 8);
#pragma unroll
      for (int i = 0; i < PR; ++i)
#pragma unroll
        for (int e = 0; e < 8; ++e) sum[i] = __builtin_fmaf(w[i].get(e), x.get(e), sum[i]);
    }
    for (int k = 512 + lane * 8; k < rank; k += 512) {
#pragma unroll
      for (int i = 0; i < PR; ++i) {
        Pack8<T> v;
        v.load(wh + min(r + i * rstep, vrows - 1) * rank + k);
#pragma unroll
        for (int e = 0; e < 8; ++e) sum[i] = __builtin_fmaf(v.get(e), lat[k + e], sum[i]);
      }
    }
    if (r + PR * rstep < vrows) load_rows(r + PR * rstep);
    float mine = 0.f;
#pragma unroll
    for (int i = 0; i < PR; ++i) {
      const float t = wave_sum(sum[i]);
      if (lane == i) mine = t;
    }
    if (lane < PR && r + lane * rstep < vrows) out[(int64_t)head * vrows + r + lane * rstep] = from_f<T>(mine);
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
