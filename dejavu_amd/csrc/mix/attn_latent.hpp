// Decode attention over a latent cache on the matrix cores: all heads share one row per token that is key and value
// (bf16 cache and queries, fp32 scores and sums).  A workgroup of NW waves takes a split of the tokens for 16 HT heads,
// 16 NW tokens at a time: wave w scores tokens 16 w .. 16 w + 15 straight from the registers that hold their cache rows, the same
// registers are written to LDS transposed (rank x tokens), and the second product reads them from there.
#pragma once
#include "attn_rows.hpp"

namespace dv {

// Position of element (r, token) in the transposed tile: rows of KT tokens in chunks of 8, the chunks permuted by the
// row so that both the transposing stores and the 16-byte reads spread over the banks.
template <int KT>
__device__ __forceinline__ int latent_swizzle(int r, int chunk) {
  return r * KT + ((chunk ^ (r & 7) ^ ((r >> 3) & 3) * 2) << 3);
}

template <int RT, int HT, int NW>
constexpr size_t latent_lds_bytes() {
  return (size_t)RT * 16 * 16 * NW * 2 + (size_t)HT * 16 * (RT * 16 + 8) * 2 + (size_t)HT * 16 * (16 * NW + 8) * 2;
}

// RT: tiles of 16 latent channels (16 RT >= rank), HT: tiles of 16 heads.  Grid: (splits, ceil(H / (16 HT))).
template <int RT, int HT, int NW>
__global__ __launch_bounds__(64 * NW) void latent_attn_kernel(AttnArgs a) {
  constexpr int KT = 16 * NW, TH = 64 * NW;  // tokens per tile, threads
  constexpr int QL = RT * 16 + 8, PL = KT + 8, ST = RT / 2, TW = RT / NW;
  static_assert(TW >= 1, "every wave owns latent channels");
  extern __shared__ __attribute__((aligned(16))) unsigned char smem_raw[];
  bf16_t* ct = reinterpret_cast<bf16_t*>(smem_raw);
  bf16_t* qs = ct + RT * 16 * KT;
  bf16_t* ps = qs + HT * 16 * QL;
  __shared__ float red[NW][HT * 16];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l16 = lane & 15, q4 = lane >> 4;
  const int h0 = blockIdx.y * HT * 16, split = blockIdx.x, rank = a.vdim_s;
  const int pos = seq_position(a.pos_dev, a.pos_host);
  const int per = ((pos + 1 + a.splits - 1) / a.splits + KT - 1) / KT * KT;
  const int j0 = split * per, j1 = min(pos + 1, j0 + per);
  const bf16_t* C = reinterpret_cast<const bf16_t*>(a.k);
  uint4_t cf[ST];
  auto fetch = [&](int jt) {
    // past the last token the weights are zero, past the last channel the queries are
    const bf16_t* row = C + (int64_t)min(jt + wave * 16 + l16, j1 - 1) * a.ldk;
#pragma unroll
    for (int s = 0; s < ST; ++s) cf[s] = *reinterpret_cast<const uint4_t*>(row + min(s * 32 + q4 * 8, rank - 8));
  };
  if (j0 < j1) fetch(j0);
  // queries as bf16, eight at a time, all of a thread's requested together
  const float* Q = reinterpret_cast<const float*>(a.q);
  constexpr int QN = (HT * 16 * RT * 2 + TH - 1) / TH;
  Pack8<float> qr[QN];
#pragma unroll
  for (int u = 0; u < QN; ++u) {
    const int i = u * TH + tid, h = i / (RT * 2), d = i % (RT * 2) * 8;
    qr[u].load(Q + (int64_t)min(h0 + h, a.H - 1) * rank + min(d, rank - 8));
  }
#pragma unroll
  for (int u = 0; u < QN; ++u) {
    const int i = u * TH + tid, h = i / (RT * 2), d = i % (RT * 2) * 8;
    bf16x8_t v;
#pragma unroll
    for (int e = 0; e < 8; ++e) v[e] = (bf16_t)(d < rank ? qr[u].get(e) : 0.f);
    if (h < HT * 16) *reinterpret_cast<bf16x8_t*>(qs + h * QL + d) = v;
  }
  float4_t o[TW][HT];
  float m[HT], l[HT];
#pragma unroll
  for (int t = 0; t < HT; ++t) {
    m[t] = -1e30f;
    l[t] = 0.f;
#pragma unroll
    for (int i = 0; i < TW; ++i) o[i][t] = float4_t{0.f, 0.f, 0.f, 0.f};
  }
  const float sc = a.scale * 1.44269504088896340736f;
  __syncthreads();
  for (int jt = j0; jt < j1; jt += KT) {
    float4_t s[HT];
#pragma unroll
    for (int t = 0; t < HT; ++t) s[t] = float4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int k = 0; k < ST; ++k)
#pragma unroll
      for (int t = 0; t < HT; ++t) {
        const bf16x8_t qf = *reinterpret_cast<const bf16x8_t*>(qs + (t * 16 + l16) * QL + k * 32 + q4 * 8);
        s[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, cf[k]), qf, s[t], 0, 0, 0);
      }
    // transposed store: neighbouring lanes hold neighbouring tokens; the even one stores the even channel of each
    // pair, the odd one the odd channel, two tokens per 32 bits
    const int tok = wave * 16 + (l16 & ~1), odd = lane & 1;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      // channel 32 k + 8 q4 + 2 e + odd; its place but for 32 k rows
      bf16_t* place = ct + latent_swizzle<KT>(q4 * 8 + 2 * e + odd, tok >> 3) + (tok & 7);
#pragma unroll
      for (int k = 0; k < ST; ++k) {
        const unsigned own = cf[k][e];
        const unsigned other = (unsigned)__builtin_amdgcn_update_dpp(0, (int)own, 0xB1, 0xf, 0xf, false);
        const unsigned v = odd ? ((other >> 16) | (own & 0xffff0000u)) : ((own & 0xffffu) | (other << 16));
        *reinterpret_cast<unsigned*>(place + k * 32 * KT) = v;
      }
    }
    if (jt + KT < j1) fetch(jt + KT);
    float c[HT];
#pragma unroll
    for (int t = 0; t < HT; ++t) {
      float mx = -INFINITY;
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const bool in = jt + wave * 16 + q4 * 4 + i < j1;
        s[t][i] = in ? s[t][i] * sc : -INFINITY;
        mx = fmaxf(mx, s[t][i]);
      }
      mx = fmaxf(mx, __shfl_xor(mx, 16, kWave));
      mx = fmaxf(mx, __shfl_xor(mx, 32, kWave));
      if (q4 == 0) red[wave][t * 16 + l16] = mx;
    }
    __syncthreads();
#pragma unroll
    for (int t = 0; t < HT; ++t) {
      const int h = t * 16 + l16;
      float m1 = m[t];
#pragma unroll
      for (int v = 0; v < NW; ++v) m1 = fmaxf(m1, red[v][h]);
      c[t] = __builtin_amdgcn_exp2f(m[t] - m1);
      m[t] = m1;
      l[t] *= c[t];
      bf16x4_t p;
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const float x = __builtin_amdgcn_exp2f(s[t][i] - m1);
        l[t] += x;
        p[i] = (bf16_t)x;
      }
      *reinterpret_cast<bf16x4_t*>(ps + h * PL + wave * 16 + q4 * 4) = p;
    }
    __syncthreads();
    bf16x8_t pf[KT / 32][HT];
#pragma unroll
    for (int k = 0; k < KT / 32; ++k)
#pragma unroll
      for (int t = 0; t < HT; ++t)
        pf[k][t] = *reinterpret_cast<const bf16x8_t*>(ps + (t * 16 + l16) * PL + k * 32 + q4 * 8);
#pragma unroll
    for (int i = 0; i < TW; ++i) {
      const int r = (wave * TW + i) * 16 + l16;
#pragma unroll
      for (int t = 0; t < HT; ++t) o[i][t] *= c[t];
#pragma unroll
      for (int k = 0; k < KT / 32; ++k) {
        const bf16x8_t cv = *reinterpret_cast<const bf16x8_t*>(ct + latent_swizzle<KT>(r, k * 4 + q4));
#pragma unroll
        for (int t = 0; t < HT; ++t) o[i][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(cv, pf[k][t], o[i][t], 0, 0, 0);
      }
    }
    __syncthreads();
  }
#pragma unroll
  for (int t = 0; t < HT; ++t) {
    l[t] += __shfl_xor(l[t], 16, kWave);
    l[t] += __shfl_xor(l[t], 32, kWave);
    if (q4 == 0) red[wave][t * 16 + l16] = l[t];
  }
  __syncthreads();
#pragma unroll
  for (int t = 0; t < HT; ++t) {
    const int h = h0 + t * 16 + l16;
    if (h >= a.H) continue;
    float* p = part_sums(a, 0, h, split);
#pragma unroll
    for (int i = 0; i < TW; ++i) {
      const int r = (wave * TW + i) * 16 + q4 * 4;
      if (r < rank) *reinterpret_cast<float4_t*>(p + r) = o[i][t];
    }
    if (wave == 0 && q4 == 0) {
      const int hl = t * 16 + l16;
      float* ml = part_ml(a, 0, h, split);
      ml[0] = m[t] * 0.69314718055994530942f;  // natural units
      float sum = 0.f;
#pragma unroll
      for (int v = 0; v < NW; ++v) sum += red[v][hl];
      ml[1] = sum;
    }
  }
}

}  // namespace dv
