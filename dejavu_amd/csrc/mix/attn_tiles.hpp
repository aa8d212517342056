// Causal softmax attention of a portion of a prompt on the matrix cores (bf16 operands, fp32 scores and sums):
// grouped key/value heads, different query/key and value sizes, optional sliding window or chunks, bias by distance,
// sink and output gate.
//
// A workgroup takes 128 queries of one head, a wave 32 of them.  Scores are computed transposed (keys x queries),
// so a lane holds the scores of ONE query: the softmax is lane-local but for one exchange between the half waves,
// and the weights are already in the operand layout of the second product when its keys are taken in the order
// the accumulator has them (key permutation 0-3, 8-11 | 4-7, 12-15 inside 16).
#pragma once
#include "attn_rows.hpp"

namespace dv {

constexpr int kTileQ = 128, kTileK = 64;

// DT: query/key tiles of 16, VT: value tiles of 32.  Grid: H * ceil(n / 128), head fastest, last queries first.
template <int DT, int VT>
__global__ __launch_bounds__(256) void attn_tiles_kernel(AttnArgs a, int keys /* rows behind k and v */) {
  constexpr int DL = DT * 16 + 8, VL = kTileK + 4;  // LDS row lengths
  __shared__ __attribute__((aligned(16))) bf16_t ks[kTileK * DL];
  __shared__ __attribute__((aligned(16))) bf16_t vs[VT * 32 * VL];
  __shared__ float rs[kTileQ + kTileK];  // biases of a tile: entry i is the distance off + q0 - k0 - (kTileK - 1) + i
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l32 = lane & 31, hh = lane >> 5;
  const int head = blockIdx.x % a.H, g = head / (a.H / a.G);
  const int nblk = (a.n + kTileQ - 1) / kTileQ;
  const int q0 = (nblk - 1 - (int)(blockIdx.x / a.H)) * kTileQ;
  const int off = a.pos_host - a.base;  // key slot of query 0
  const bf16_t* K = reinterpret_cast<const bf16_t*>(a.k) + (int64_t)g * a.k_head;
  const bf16_t* V = reinterpret_cast<const bf16_t*>(a.v) + (int64_t)g * a.v_head;

  const int qi = q0 + wave * 32 + l32;  // this lane's query
  bf16x8_t qf[DT];
  {
    const bf16_t* q = reinterpret_cast<const bf16_t*>(a.q) + (int64_t)(qi < a.n ? qi : 0) * a.ldq + (int64_t)head * a.dim_s;
#pragma unroll
    for (int t = 0; t < DT; ++t) {
      const int d = t * 16 + hh * 8;
      uint4_t z = {0, 0, 0, 0};
      if (qi < a.n && d < a.dim_s) z = *reinterpret_cast<const uint4_t*>(q + d);
      qf[t] = __builtin_bit_cast(bf16x8_t, z);
    }
  }
  const int qslot = off + qi;
  auto oldest_slot = [&](int q) { return max(0, oldest_key(a, a.pos_host + q) - a.base); };
  const int klo = oldest_slot(min(qi, a.n - 1));
  const int wklo = __builtin_amdgcn_readfirstlane(klo);
  const int wkhi = oldest_slot(min(q0 + wave * 32 + 31, a.n - 1));
  const int wlo = off + q0 + wave * 32, whi = min(off + q0 + wave * 32 + 31, off + a.n - 1);  // slots of the wave
  const int bhi = min(off + q0 + kTileQ - 1, off + a.n - 1);
  const int first = oldest_slot(q0) / kTileK * kTileK;
  const float* rel = a.rel ? a.rel + (int64_t)head * a.rel_len : nullptr;
  constexpr float kLog2e = 1.44269504088896340736f;
  const float rel_far = rel ? rel[a.rel_len - 1] * kLog2e : 0.f;
  float rr = 0.f;
  const int last = bhi;

  constexpr int KV = (kTileK * DT * 2 + 255) / 256;       // 16-byte loads of K per thread
  constexpr int VV = (kTileK / 2 * VT * 4 + 255) / 256;   // pairs of 16-byte loads of V per thread
  uint4_t kr[KV], vr[VV][2];
  auto fetch = [&](int k0) {
    if (rel) rr = rel[min(max(off + q0 - k0 - (kTileK - 1) + tid, 0), a.rel_len - 1)] * kLog2e;
    // past the last key the weights are zero; past the last channel the queries are, or nothing is stored
#pragma unroll
    for (int i = 0; i < KV; ++i) {
      const int at = i * 256 + tid, r = at / (DT * 2), d = at % (DT * 2) * 8;
      kr[i] = *reinterpret_cast<const uint4_t*>(K + (int64_t)min(k0 + r, keys - 1) * a.ldk + min(d, a.dim_s - 8));
    }
#pragma unroll
    for (int i = 0; i < VV; ++i) {
      const int at = i * 256 + tid, r = at % (kTileK / 2) * 2, d = min(at / (kTileK / 2) * 8, a.vdim_s - 8);
      vr[i][0] = *reinterpret_cast<const uint4_t*>(V + (int64_t)min(k0 + r, keys - 1) * a.ldv + d);
      vr[i][1] = *reinterpret_cast<const uint4_t*>(V + (int64_t)min(k0 + r + 1, keys - 1) * a.ldv + d);
    }
  };
  auto put = [&]() {
    if (rel && tid < kTileQ + kTileK) rs[tid] = rr;
#pragma unroll
    for (int i = 0; i < KV; ++i) {
      const int at = i * 256 + tid, r = at / (DT * 2), d = at % (DT * 2) * 8;
      if (r < kTileK) *reinterpret_cast<uint4_t*>(&ks[r * DL + d]) = kr[i];
    }
#pragma unroll
    for (int i = 0; i < VV; ++i) {
      const int at = i * 256 + tid, r = at % (kTileK / 2) * 2, d = at / (kTileK / 2) * 8;
      if (d < VT * 32) {
#pragma unroll
        for (int e = 0; e < 4; ++e) {  // two keys of a value channel side by side
          const unsigned x = vr[i][0][e], y = vr[i][1][e];
          *reinterpret_cast<unsigned*>(&vs[(d + 2 * e) * VL + r]) = (x & 0xffffu) | (y << 16);
          *reinterpret_cast<unsigned*>(&vs[(d + 2 * e + 1) * VL + r]) = (x >> 16) | (y & 0xffff0000u);
        }
      }
    }
  };

  float16_t o[VT];
#pragma unroll
  for (int t = 0; t < VT; ++t)
#pragma unroll
    for (int i = 0; i < 16; ++i) o[t][i] = 0.f;
  float m = -1e30f, l = 0.f;  // l: this half wave's share
  const float sc = a.scale * kLog2e;

  fetch(first);
  for (int k0 = first; k0 <= last; k0 += kTileK) {
    __syncthreads();
    put();
    __syncthreads();
    if (k0 + kTileK <= last) fetch(k0 + kTileK);
    const bool seen = k0 <= whi && k0 + kTileK - 1 >= wklo;
    if (!seen) continue;
    float16_t s[2];
#pragma unroll
    for (int kt = 0; kt < 2; ++kt) {
#pragma unroll
      for (int i = 0; i < 16; ++i) s[kt][i] = 0.f;
#pragma unroll
      for (int t = 0; t < DT; ++t) {
        const bf16x8_t kf = *reinterpret_cast<const bf16x8_t*>(&ks[(kt * 32 + l32) * DL + t * 16 + hh * 8]);
        s[kt] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(kf, qf[t], s[kt], 0, 0, 0);
      }
    }
    const bool full = k0 + kTileK - 1 <= wlo && k0 >= wkhi;
    if (rel && wlo - (k0 + kTileK - 1) < a.rel_len - 1) {
      const float* rp = rs + wave * 32 + l32 + kTileK - 1 - 4 * hh;
#pragma unroll
      for (int kt = 0; kt < 2; ++kt)
#pragma unroll
        for (int i = 0; i < 16; ++i) s[kt][i] = __builtin_fmaf(s[kt][i], sc, rp[-(kt * 32 + 8 * (i >> 2) + (i & 3))]);
    } else {  // no bias, or one for all
#pragma unroll
      for (int kt = 0; kt < 2; ++kt)
#pragma unroll
        for (int i = 0; i < 16; ++i) s[kt][i] = __builtin_fmaf(s[kt][i], sc, rel_far);
    }
    float mx = -INFINITY;
#pragma unroll
    for (int kt = 0; kt < 2; ++kt)
#pragma unroll
      for (int i = 0; i < 16; ++i) {
        float x = s[kt][i];
        if (!full) {
          const int key = k0 + kt * 32 + 8 * (i >> 2) + 4 * hh + (i & 3);
          if (key > qslot || key < klo) x = -INFINITY;
        }
        s[kt][i] = x;
        mx = fmaxf(mx, x);
      }
    mx = fmaxf(mx, __shfl_xor(mx, 32, kWave));
    const float m1 = fmaxf(m, mx);
    const float c = __builtin_amdgcn_exp2f(m - m1);
    m = m1;
    l *= c;
#pragma unroll
    for (int kt = 0; kt < 2; ++kt)
#pragma unroll
      for (int i = 0; i < 16; ++i) {
        const float p = __builtin_amdgcn_exp2f(s[kt][i] - m1);
        s[kt][i] = p;
        l += p;
      }
#pragma unroll
    for (int t = 0; t < VT; ++t)
#pragma unroll
      for (int i = 0; i < 16; ++i) o[t][i] *= c;
#pragma unroll
    for (int ks4 = 0; ks4 < 4; ++ks4) {
      bf16x8_t pf;
#pragma unroll
      for (int e = 0; e < 8; ++e) pf[e] = (bf16_t)s[ks4 >> 1][8 * (ks4 & 1) + e];
#pragma unroll
      for (int t = 0; t < VT; ++t) {
        const bf16_t* vp = &vs[(t * 32 + l32) * VL + ks4 * 16 + 4 * hh];
        uint4_t w;
        const uint2_t w0 = *reinterpret_cast<const uint2_t*>(vp), w1 = *reinterpret_cast<const uint2_t*>(vp + 8);
        w[0] = w0[0];
        w[1] = w0[1];
        w[2] = w1[0];
        w[3] = w1[1];
        o[t] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(bf16x8_t, w), pf, o[t], 0, 0, 0);
      }
    }
  }
  l += __shfl_xor(l, 32, kWave);
  if (qi >= a.n) return;
  m *= 0.69314718055994530942f;  // back to natural units
  float c;
  const float f = attn_factor<bf16_t>(a, qi, head, m, l, &c) * c;
  bf16_t* out = reinterpret_cast<bf16_t*>(a.out) + ((int64_t)qi * a.H + head) * a.vdim_s;
#pragma unroll
  for (int t = 0; t < VT; ++t)
#pragma unroll
    for (int i = 0; i < 16; i += 4) {
      const int d = t * 32 + 2 * i + 4 * hh;
      if (d < a.vdim_s) {
        bf16x4_t w = {(bf16_t)(o[t][i] * f), (bf16_t)(o[t][i + 1] * f), (bf16_t)(o[t][i + 2] * f), (bf16_t)(o[t][i + 3] * f)};
        *reinterpret_cast<bf16x4_t*>(out + d) = w;
      }
    }
}

}  // namespace dv
