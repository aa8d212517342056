// Element types of the mixer kernels (bf16 or fp32 storage, fp32 arithmetic) and small wave helpers.
#pragma once
#include "../../../include/dejavu_mixers.h"
#include "../common.hpp"

namespace dv {

typedef __bf16 bf16_t;
typedef __bf16 bf16x4_t __attribute__((ext_vector_type(4)));
typedef __bf16 bf16x8_t __attribute__((ext_vector_type(8)));
typedef unsigned uint4_t __attribute__((ext_vector_type(4)));
typedef unsigned uint2_t __attribute__((ext_vector_type(2)));

// Eight consecutive elements as loaded from memory (16 or 32 bytes).
template <typename T>
struct Pack8;
template <>
struct Pack8<bf16_t> {
  uint4_t v;
  __device__ __forceinline__ void load(const bf16_t* p) { v = *reinterpret_cast<const uint4_t*>(p); }
  __device__ __forceinline__ void load_stream(const bf16_t* p) {
    v = __builtin_nontemporal_load(reinterpret_cast<const uint4_t*>(p));
  }
  __device__ __forceinline__ void zero() { v = uint4_t{0, 0, 0, 0}; }
  // element e of 0..7 as fp32 (bf16 is the upper half of an fp32)
  __device__ __forceinline__ float get(int e) const {
    const unsigned w = v[e >> 1];
    return __uint_as_float((e & 1) ? (w & 0xffff0000u) : (w << 16));
  }
};
template <>
struct Pack8<float> {
  float4_t a, b;
  __device__ __forceinline__ void load(const float* p) {
    a = *reinterpret_cast<const float4_t*>(p);
    b = *reinterpret_cast<const float4_t*>(p + 4);
  }
  __device__ __forceinline__ void load_stream(const float* p) {
    a = __builtin_nontemporal_load(reinterpret_cast<const float4_t*>(p));
    b = __builtin_nontemporal_load(reinterpret_cast<const float4_t*>(p + 4));
  }
  __device__ __forceinline__ void zero() { a = b = float4_t{0.f, 0.f, 0.f, 0.f}; }
  __device__ __forceinline__ float get(int e) const { return e < 4 ? a[e] : b[e - 4]; }
};

__device__ __forceinline__ float to_f(float v) { return v; }
__device__ __forceinline__ float to_f(bf16_t v) { return (float)v; }
template <typename T>
__device__ __forceinline__ T from_f(float v) { return (T)v; }

// Four consecutive values in the storage type.
template <typename T>
__device__ __forceinline__ void store_quad(T* p, const float4_t& v) {
  typedef T quad_t __attribute__((ext_vector_type(4)));
  *reinterpret_cast<quad_t*>(p) = quad_t{from_f<T>(v[0]), from_f<T>(v[1]), from_f<T>(v[2]), from_f<T>(v[3])};
}
template <typename T>
__device__ __forceinline__ float4_t load_quad(const T* p) {
  typedef T quad_t __attribute__((ext_vector_type(4)));
  const quad_t v = *reinterpret_cast<const quad_t*>(p);
  return float4_t{to_f(v[0]), to_f(v[1]), to_f(v[2]), to_f(v[3])};
}

// Sum over the 16 lanes of a DPP row; every lane ends with the total.
template <int CTRL>
__device__ __forceinline__ float dpp_add(float v) {
  const int o = __builtin_amdgcn_update_dpp(0, __float_as_int(v), CTRL, 0xf, 0xf, false);
  return v + __int_as_float(o);
}
__device__ __forceinline__ float row16_sum(float v) {
  v = dpp_add<0xB1>(v);   // quad_perm 1,0,3,2
  v = dpp_add<0x4E>(v);   // quad_perm 2,3,0,1
  v = dpp_add<0x141>(v);  // row_half_mirror: the other quad of the half row
  return dpp_add<0x140>(v);  // row_mirror: the other half row
}
// Sum over the wave; every lane ends with the total.
__device__ __forceinline__ float wave_sum(float v) {
  v = row16_sum(v);
  v += __shfl_xor(v, 16, kWave);
  return v + __shfl_xor(v, 32, kWave);
}

// fp32 exponential from the hardware's base-2 one: x log2(e) is kept in two parts, the second as a correction of the
// result.  Arguments are held where the result is finite.
__device__ __forceinline__ float exp_f(float x) {
  x = fminf(fmaxf(x, -104.f), 88.5f);
  const float hi = x * 1.44269504f;
  const float lo = __builtin_fmaf(x, 1.92596299e-8f, __builtin_fmaf(x, 1.44269504f, -hi));
  const float r = __builtin_amdgcn_exp2f(hi);
  return __builtin_fmaf(r, lo * 0.693147181f, r);
}
__device__ __forceinline__ float rcp_f(float x) { return __builtin_amdgcn_rcpf(x); }
__device__ __forceinline__ float sigmoid_f(float z) { return rcp_f(1.f + exp_f(-z)); }
__device__ __forceinline__ float silu_f(float z) { return z * sigmoid_f(z); }
// log(1 + e), 0 <= e <= 1: the Taylor series where 1 + e would lose the digits of e
__device__ __forceinline__ float log1p_f(float e) {
  const float series = e * (1.f - e * (0.5f - e * (0.333333333f - e * 0.25f)));
  return e < 0.015625f ? series : __logf(1.f + e);
}
__device__ __forceinline__ float softplus_f(float z) { return fmaxf(z, 0.f) + log1p_f(exp_f(-fabsf(z))); }
__device__ __forceinline__ float tanh_f(float x) {
  const float t = exp_f(-2.f * fabsf(x)), x2 = x * x;
  const float big = copysignf((1.f - t) * rcp_f(1.f + t), x);
  const float series = x * (1.f - x2 * (0.333333333f - x2 * (0.133333333f - x2 * 0.0539682540f)));
  return x2 < 0.01f ? series : big;
}

// Dynamic tanh: tanh(alpha x) w + b, per channel.
using DynTanh = dvDynTanh;
__device__ __forceinline__ float dyn_tanh(float x, const DynTanh& n, int c) {
  return __builtin_fmaf(tanh_f(n.alpha * x), n.w[c], n.b[c]);
}

// Loads below are unconditional from clamped addresses wherever a bound can be met (what lies past it is masked where
// it is used): a guarded load becomes a branch, and a row of branches keeps few loads in flight.

// The sequence position of a call: on the device (captured decode steps) or passed by the host.
__device__ __forceinline__ int seq_position(const int* dev, int host) { return dev ? *dev : host; }

}  // namespace dv
