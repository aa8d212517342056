// C ABI of libdejavu_mixers.so (include/dejavu_mixers.h): argument checks on the host, then launches.
#include "../../include/dejavu_mixers.h"

#include <hip/hip_runtime.h>

#include <atomic>

#include "mix/attn_latent.hpp"
#include "mix/attn_rows.hpp"
#include "mix/attn_tiles.hpp"
#include "mix/delta_rule.hpp"
#include "mix/hyper.hpp"
#include "mix/linear_rows.hpp"
#include "mix/linear_tiles.hpp"
#include "mix/short_conv.hpp"
#include "mix/ssd.hpp"
#include "mix/stream.hpp"

using namespace dv;

namespace {

inline bool al16(const void* p) { return (reinterpret_cast<uintptr_t>(p) & 15u) == 0; }
inline int launched() { return hipGetLastError() == hipSuccess ? DV_OK : DV_ERR_LAUNCH; }
inline hipStream_t st(void* s) { return reinterpret_cast<hipStream_t>(s); }
inline bool dtype_ok(int d) { return d == DV_BF16 || d == DV_F32; }
inline unsigned blocks_of(int64_t work, int64_t per) { return (unsigned)((work + per - 1) / per); }

// Dynamic LDS above 48 KiB is granted per kernel and device.
template <auto KERNEL>
int grant(size_t bytes) {
  static std::atomic<size_t> granted[64];
  if (bytes <= 48 * 1024) return DV_OK;
  if (bytes > 158 * 1024) return DV_ERR_UNSUPPORTED;
  int dev = 0;
  if (hipGetDevice(&dev) != hipSuccess || dev < 0 || dev >= 64) return DV_ERR_UNSUPPORTED;
  if (bytes <= granted[dev].load(std::memory_order_relaxed)) return DV_OK;
  if (hipFuncSetAttribute(reinterpret_cast<const void*>(KERNEL), hipFuncAttributeMaxDynamicSharedMemorySize, (int)bytes) !=
      hipSuccess)
    return DV_ERR_UNSUPPORTED;
  granted[dev].store(bytes, std::memory_order_relaxed);
  return DV_OK;
}

template <auto KERNEL, typename... A>
int launch_lds(dim3 grid, dim3 block, size_t lds, hipStream_t s, A... args) {
  const int rc = grant<KERNEL>(lds);
  if (rc != DV_OK) return rc;
  hipLaunchKernelGGL(KERNEL, grid, block, lds, s, args...);
  return launched();
}

// ---- one row ---------------------------------------------------------------
template <typename T, int BEFORE, int AFTER>
int linear_row(const RowsArgs& a, hipStream_t s) {
  constexpr int R = 2, U = sizeof(T) == 2 ? 4 : 2;
  const int ntasks = (a.M + R - 1) / R;
  int blocks = (ntasks + 3) / 4;
  if (blocks > 2048) blocks = 2048;
  if (a.side_x) ++blocks;
  return launch_lds<linear_rows_kernel<T, BEFORE, AFTER, R, U>>(dim3(blocks), dim3(256), (size_t)a.K * sizeof(T), s, a);
}
template <typename T>
int linear_row_any(int before, int after, const RowsArgs& a, hipStream_t s) {
  if (before == DV_ROW_PLAIN) {
    switch (after) {
      case DV_OUT_F32: return linear_row<T, DV_ROW_PLAIN, DV_OUT_F32>(a, s);
      case DV_OUT_T: return linear_row<T, DV_ROW_PLAIN, DV_OUT_T>(a, s);
      case DV_OUT_GLU: return linear_row<T, DV_ROW_PLAIN, DV_OUT_GLU>(a, s);
      case DV_OUT_RESIDUAL: return linear_row<T, DV_ROW_PLAIN, DV_OUT_RESIDUAL>(a, s);
      case DV_OUT_CONV: return linear_row<T, DV_ROW_PLAIN, DV_OUT_CONV>(a, s);
      case DV_OUT_HYPER: return linear_row<T, DV_ROW_PLAIN, DV_OUT_HYPER>(a, s);
    }
  } else if (before == DV_ROW_RMS) {
    switch (after) {
      case DV_OUT_F32: return linear_row<T, DV_ROW_RMS, DV_OUT_F32>(a, s);
      case DV_OUT_GLU: return linear_row<T, DV_ROW_RMS, DV_OUT_GLU>(a, s);
      case DV_OUT_CONV: return linear_row<T, DV_ROW_RMS, DV_OUT_CONV>(a, s);
    }
  } else if (before == DV_ROW_GROUPS && after == DV_OUT_HYPER) {
    return linear_row<T, DV_ROW_GROUPS, DV_OUT_HYPER>(a, s);
  } else if (before == DV_ROW_GROUPS && after == DV_OUT_T) {
    return linear_row<T, DV_ROW_GROUPS, DV_OUT_T>(a, s);
  } else if (before == DV_ROW_HEADS && after == DV_OUT_RESIDUAL) {
    return linear_row<T, DV_ROW_HEADS, DV_OUT_RESIDUAL>(a, s);
  }
  return DV_ERR_UNSUPPORTED;
}

// ---- short convolution -------------------------------------------------------
template <typename T, typename TO, int LPH>
int short_conv_lanes(const ConvArgs& a, int heads, hipStream_t s) {
  const dim3 grid(blocks_of(heads, 256 / LPH), blocks_of(a.n, kConvTokens));
  switch (a.taps) {
    case 1: hipLaunchKernelGGL((short_conv_kernel<T, TO, LPH, 1>), grid, dim3(256), 0, s, a); break;
    case 2: hipLaunchKernelGGL((short_conv_kernel<T, TO, LPH, 2>), grid, dim3(256), 0, s, a); break;
    case 3: hipLaunchKernelGGL((short_conv_kernel<T, TO, LPH, 3>), grid, dim3(256), 0, s, a); break;
    default: hipLaunchKernelGGL((short_conv_kernel<T, TO, LPH, 4>), grid, dim3(256), 0, s, a); break;
  }
  return launched();
}
template <typename T, typename TO>
int short_conv_types(const ConvArgs& a, int heads, int widest, hipStream_t s) {
  if (a.taps > 4 || widest > 512 || (a.n + kConvTokens - 1) / kConvTokens > 65535) {
    hipLaunchKernelGGL((short_conv_any_kernel<T, TO>), dim3(blocks_of((int64_t)a.n * heads, 4)), dim3(256), 0, s, a);
    return launched();
  }
  if (widest <= 8) return short_conv_lanes<T, TO, 1>(a, heads, s);
  if (widest <= 64) return short_conv_lanes<T, TO, 8>(a, heads, s);
  if (widest <= 128) return short_conv_lanes<T, TO, 16>(a, heads, s);
  if (widest <= 256) return short_conv_lanes<T, TO, 32>(a, heads, s);
  return short_conv_lanes<T, TO, 64>(a, heads, s);
}

// ---- attention rows --------------------------------------------------------
template <typename T, typename TQ, int RH>
int attn_rows_rh(const AttnArgs& a, hipStream_t s) {
  const int rep = a.H / a.G;
  const dim3 grid(a.splits, a.G * ((rep + RH - 1) / RH), a.n);
  const size_t lds = (size_t)RH * a.dim_s * 4 + (size_t)attn_red_floats(RH, a.vdim_s) * 4 + (size_t)(a.dim_s + a.vdim_s) * sizeof(T);
  return launch_lds<attn_rows_kernel<T, TQ, RH>>(grid, dim3(256), lds, s, a);
}
template <typename T, typename TQ>
int attn_rows_any(const AttnArgs& a, hipStream_t s) {
  const int rep = a.H / a.G;
  if (rep >= 8) return attn_rows_rh<T, TQ, 8>(a, s);
  if (rep >= 3) return attn_rows_rh<T, TQ, 4>(a, s);
  if (rep == 2) return attn_rows_rh<T, TQ, 2>(a, s);
  return attn_rows_rh<T, TQ, 1>(a, s);
}

// ---- delta rule --------------------------------------------------------------
constexpr int kDeltaSegment = 4096;  // tokens whose chunk blocks are in memory at a time
template <int NT>
int delta_scan(const DeltaArgs& a, hipStream_t s) {
  const size_t need = (size_t)((a.n < kDeltaSegment ? a.n : kDeltaSegment) + kDeltaChunk - 1) / kDeltaChunk * a.heads *
                      DeltaChunk<NT>::floats;
  if ((size_t)a.tm_floats < need) return DV_ERR_WORKSPACE;
  for (int t0 = 0; t0 < a.n; t0 += kDeltaSegment) {
    DeltaArgs b = a;
    b.q += (int64_t)t0 * a.kv_heads * a.dim_s;
    b.k += (int64_t)t0 * a.kv_heads * a.dim_s;
    b.v += (int64_t)t0 * a.heads * a.vdim_s;
    b.g += (int64_t)t0 * a.heads * a.dim_s;
    b.o += (int64_t)t0 * a.heads * a.vdim_s;
    b.beta += (int64_t)t0 * a.heads;
    b.n = a.n - t0 < kDeltaSegment ? a.n - t0 : kDeltaSegment;
    int rc = launch_lds<delta_chunk_kernel<NT>>(dim3(a.heads, (b.n + kDeltaChunk - 1) / kDeltaChunk), dim3(256),
                                                (size_t)3 * kDeltaChunk * 64 * NT * 4, s, b);
    if (rc != DV_OK) return rc;
    rc = launch_lds<delta_scan_kernel<NT>>(dim3((unsigned)(a.heads * ((a.vdim_s + kDeltaCols - 1) / kDeltaCols))),
                                           dim3(256), 0, s, b);
    if (rc != DV_OK) return rc;
  }
  return DV_OK;
}

template <int RT, int HT>
int latent_heads(const AttnArgs& a, hipStream_t s) {
  constexpr int NW = RT >= 8 ? 8 : 4;
  return launch_lds<latent_attn_kernel<RT, HT, NW>>(dim3(a.splits, (a.H + 16 * HT - 1) / (16 * HT)), dim3(64 * NW),
                                                    latent_lds_bytes<RT, HT, NW>(), s, a);
}
// Sixteen heads per workgroup; with many heads (workgroups enough without it) and room in LDS 32, so that the cache is
// read half as often.
template <int RT>
int latent_tiles(const AttnArgs& a, hipStream_t s) {
  if constexpr (RT <= 16) {
    if (a.splits * ((a.H + 15) / 16) > 512) return latent_heads<RT, 2>(a, s);
  }
  return latent_heads<RT, 1>(a, s);
}

int attn_args_ok(const AttnArgs* a) {
  if (!a || !a->q || !a->k || !a->v || a->n < 1 || a->H < 1 || a->G < 1 || a->H % a->G || a->dim_s < 8 ||
      a->vdim_s < 8 || a->splits < 1 || a->splits > kMaxSplits || (a->splits > 1 && !a->part) || (a->splits == 1 && !a->out) ||
      (!a->fresh_k != !a->fresh_v) || a->window < 0 || a->chunk < 0 || (a->window > 0 && a->chunk > 0) ||
      (a->rel && a->rel_len < 1) || (a->other_v && (!a->lambda || !a->fresh_v)) || ((a->q_w || a->k_w) && a->norm_dim < 1))
    return DV_ERR_INVALID_ARG;
  if (a->dim_s % 8 || a->vdim_s % 8 || a->ldk % 8 || a->ldv % 8 || a->k_head % 8 || a->v_head % 8 || !al16(a->k) ||
      !al16(a->v) || !al16(a->q))
    return DV_ERR_ALIGNMENT;
  if (a->vdim_s > 2048 || a->n > 65535 || (int64_t)a->H > 65535) return DV_ERR_UNSUPPORTED;
  return DV_OK;
}

// ---- residual streams ------------------------------------------------------------
int hyper_ok(const dvHyper* r, const dvRmsOut* norm) {
  if (!r || !r->x || r->streams < 1 || r->streams > DV_HYPER_MAX || r->width < 4 || !norm || (!r->u && !norm->h) ||
      (norm->h && (!norm->w || norm->dim < 1 || norm->dim > r->width)))
    return DV_ERR_INVALID_ARG;
  if (r->width % 8 || !al16(r->x) || !al16(r->u) || !al16(norm->h) || !al16(norm->w)) return DV_ERR_ALIGNMENT;
  return DV_OK;
}
template <typename T, int SM, bool EMBED>
int hyper_rows(const void* y, int n, const dvHyper& r, const dvEmbedArgs& e, const dvRmsOut& norm, hipStream_t s) {
  const dim3 grid(n, norm.h ? 1 : (r.width + 1023) / 1024);
  const size_t lds = norm.h ? (size_t)r.width * 4 : 0;
  if (norm.h && n <= 512 && r.width > 1024)  // few rows: more threads for each
    return launch_lds<hyper_rows_kernel<T, SM, EMBED, 1024>>(grid, dim3(1024), lds, s, (const T*)y, r, e, norm);
  return launch_lds<hyper_rows_kernel<T, SM, EMBED, 256>>(grid, dim3(256), lds, s, (const T*)y, r, e, norm);
}

// ---- Mamba-2 -----------------------------------------------------------------------
constexpr int kSsdSegment = 4096;  // tokens whose chunk blocks are in memory at a time
template <typename T, int NT>
int ssd_scan(const SsdArgs& a, hipStream_t s) {
  const size_t need = (size_t)((a.n < kSsdSegment ? a.n : kSsdSegment) + kSsdChunk - 1) / kSsdChunk * a.heads * SsdChunk::floats;
  if ((size_t)a.tm_floats < need) return DV_ERR_WORKSPACE;
  const int rep = a.heads / a.groups;
  for (int t0 = 0; t0 < a.n; t0 += kSsdSegment) {
    SsdArgs b = a;
    b.xbc += (int64_t)t0 * a.ld;
    b.dt = reinterpret_cast<const T*>(a.dt) + (int64_t)t0 * a.lddt;
    b.y += (int64_t)t0 * a.ldy;
    b.n = a.n - t0 < kSsdSegment ? a.n - t0 : kSsdSegment;
    const int chunks = (b.n + kSsdChunk - 1) / kSsdChunk;
    int hp = 1;  // heads per workgroup: as many as leave four workgroups per compute unit
    while (hp < rep && (int64_t)a.heads * chunks / (2 * hp) >= 1024) hp *= 2;
    if (hp > rep) hp = rep;
    hipLaunchKernelGGL((ssd_chunk_kernel<T>), dim3((unsigned)(a.groups * ((rep + hp - 1) / hp)), chunks), dim3(256), 0, s, b, hp);
    int rc = launched();
    if (rc != DV_OK) return rc;
    // 32 columns per workgroup read B, C and M half as often, if that leaves about a workgroup per compute unit (and
    // the operands of two chunks fit the registers)
    constexpr int TC = NT <= 2 ? 2 : 1;
    const int wide = (a.vdim + TC * kSsdCols - 1) / (TC * kSsdCols), narrow = (a.vdim + kSsdCols - 1) / kSsdCols;
    if (a.vdim % TC == 0 && a.heads * wide >= 192)
      hipLaunchKernelGGL((ssd_scan_kernel<NT, TC>), dim3((unsigned)(a.heads * wide)), dim3(256), 0, s, b);
    else
      hipLaunchKernelGGL((ssd_scan_kernel<NT, 1>), dim3((unsigned)(a.heads * narrow)), dim3(256), 0, s, b);
    rc = launched();
    if (rc != DV_OK) return rc;
  }
  return DV_OK;
}
template <typename T>
int ssd_scan_any(const SsdArgs& a, hipStream_t s) {
  if (a.state_s <= 64) return ssd_scan<T, 1>(a, s);
  if (a.state_s <= 128) return ssd_scan<T, 2>(a, s);
  if (a.state_s <= 256) return ssd_scan<T, 4>(a, s);
  return DV_ERR_UNSUPPORTED;
}

template <int DT, int VT>
int attn_tiles_launch(const AttnArgs& a, int keys, hipStream_t s) {
  hipLaunchKernelGGL((attn_tiles_kernel<DT, VT>), dim3((unsigned)((int64_t)a.H * ((a.n + kTileQ - 1) / kTileQ))), dim3(256), 0, s, a, keys);
  return launched();
}

}  // namespace

extern "C" {

int dv_mix_embed(int dtype, const void* tokens, int64_t vocab, const void* embed, int n, int width, float* x, float* x0,
                 const dvDynTanh* norm, void* h, void* stream) {
  if (!dtype_ok(dtype) || !tokens || !embed || n < 1 || width < 1 || !x || !norm || !norm->w || !norm->b || !h)
    return DV_ERR_INVALID_ARG;
  if (width % 8 || !al16(embed) || !al16(x) || !al16(x0) || !al16(h)) return DV_ERR_ALIGNMENT;
  const int64_t* t = reinterpret_cast<const int64_t*>(tokens);
  const dim3 grid(n, (width + 2047) / 2048);
  if (dtype == DV_BF16)
    hipLaunchKernelGGL((embed_norm_kernel<bf16_t>), grid, dim3(256), 0, st(stream), t, vocab, (const bf16_t*)embed,
                       width, x, x0, *norm, (bf16_t*)h);
  else
    hipLaunchKernelGGL((embed_norm_kernel<float>), grid, dim3(256), 0, st(stream), t, vocab, (const float*)embed,
                       width, x, x0, *norm, (float*)h);
  return launched();
}

int dv_mix_residual(int dtype, const void* y, int64_t n, int width, const dvResidual* r, void* stream) {
  if (!dtype_ok(dtype) || n < 1 || width < 1 || !r || !r->x || (y && (!r->post.w || !r->post.b)) ||
      (r->h && (!r->pre.w || !r->pre.b)))
    return DV_ERR_INVALID_ARG;
  if (width % 8 || !al16(r->x) || !al16(y) || !al16(r->h)) return DV_ERR_ALIGNMENT;
  const int64_t count = n * width / 4;
  unsigned grid = blocks_of(count, 256);
  if (grid > 8192) grid = 8192;
  if (dtype == DV_BF16)
    hipLaunchKernelGGL((residual_norm_kernel<bf16_t>), dim3(grid), dim3(256), 0, st(stream), (const bf16_t*)y, count, width, *r);
  else
    hipLaunchKernelGGL((residual_norm_kernel<float>), dim3(grid), dim3(256), 0, st(stream), (const float*)y, count, width, *r);
  return launched();
}

int dv_mix_glu(int dtype, const void* gu, int64_t count, int act, float limit, void* y, void* stream) {
  if (!dtype_ok(dtype) || !gu || !y || count < 4 || (act != DV_GLU_CLAMPED && act != DV_GLU_RELU)) return DV_ERR_INVALID_ARG;
  if (count % 4 || !al16(gu)) return DV_ERR_ALIGNMENT;
  const dim3 grid(blocks_of(count, 1024));
#define DV_GLU(T)                                                                                                          \
  do {                                                                                                                     \
    if (act == DV_GLU_RELU)                                                                                                \
      hipLaunchKernelGGL((glu_kernel<T, DV_GLU_RELU>), grid, dim3(256), 0, st(stream), (const T*)gu, count, limit, (T*)y);    \
    else                                                                                                                   \
      hipLaunchKernelGGL((glu_kernel<T, DV_GLU_CLAMPED>), grid, dim3(256), 0, st(stream), (const T*)gu, count, limit, (T*)y); \
  } while (0)
  if (dtype == DV_BF16) DV_GLU(bf16_t);
  else DV_GLU(float);
#undef DV_GLU
  return launched();
}

int dv_mix_hyper_embed(int dtype, const dvEmbedArgs* e, const dvHyper* r, const dvRmsOut* norm, void* stream) {
  if (!dtype_ok(dtype) || !e || !e->tokens || !e->history || !e->embed || e->n < 1 || e->vocab < 1 || e->capacity < 1 ||
      (e->bigram && e->buckets < 1) || (!e->pos_dev && (e->pos_host < 0 || e->pos_host + (int64_t)e->n > e->capacity)))
    return DV_ERR_INVALID_ARG;
  int rc = hyper_ok(r, norm);
  if (rc != DV_OK) return rc;
  if (!r->in) return DV_ERR_INVALID_ARG;
  if (!al16(e->embed) || !al16(e->bigram)) return DV_ERR_ALIGNMENT;
  return dtype == DV_BF16 ? hyper_rows<bf16_t, 16, true>(nullptr, e->n, *r, *e, *norm, st(stream))
                          : hyper_rows<float, 16, true>(nullptr, e->n, *r, *e, *norm, st(stream));
}

int dv_mix_hyper_rows(int dtype, const void* y, int n, const dvHyper* r, const dvRmsOut* norm, void* stream) {
  if (!dtype_ok(dtype) || n < 1) return DV_ERR_INVALID_ARG;
  int rc = hyper_ok(r, norm);
  if (rc != DV_OK) return rc;
  if (!r->in || (y && (!r->mix || !r->out))) return DV_ERR_INVALID_ARG;
  if (!al16(y)) return DV_ERR_ALIGNMENT;
  const dvEmbedArgs none = {};
  if (dtype == DV_BF16)
    return r->streams <= 4 ? hyper_rows<bf16_t, 4, false>(y, n, *r, none, *norm, st(stream))
                           : hyper_rows<bf16_t, 16, false>(y, n, *r, none, *norm, st(stream));
  return r->streams <= 4 ? hyper_rows<float, 4, false>(y, n, *r, none, *norm, st(stream))
                         : hyper_rows<float, 16, false>(y, n, *r, none, *norm, st(stream));
}

int dv_mix_head_rows(int dtype, const dvHeadArgs* a, void* stream) {
  if (!dtype_ok(dtype) || !a || !a->in || a->n < 1) return DV_ERR_INVALID_ARG;
  if (a->ldi % 8 || !al16(a->in)) return DV_ERR_ALIGNMENT;
  int heads = 0;
  for (const dvHeadGroup& g : a->g) {
    if (g.heads < 0) return DV_ERR_INVALID_ARG;
    if (g.heads == 0) continue;
    if (!g.out || g.stride < 8 || g.dim < 1 || g.dim > g.stride || (g.other && (g.w || !g.lambda))) return DV_ERR_INVALID_ARG;
    if (g.stride % 8 || g.ld % 8 || !al16(g.out) || (g.other && (g.ldo % 8 || !al16(g.other)))) return DV_ERR_ALIGNMENT;
    heads += g.heads;
  }
  if (heads == 0) return DV_ERR_INVALID_ARG;
  if ((int64_t)a->n * heads >= (int64_t)1 << 31) return DV_ERR_UNSUPPORTED;
  const dim3 grid(blocks_of((int64_t)a->n * heads, 16));
  if (dtype == DV_BF16) hipLaunchKernelGGL((head_rows_kernel<bf16_t>), grid, dim3(256), 0, st(stream), *a);
  else hipLaunchKernelGGL((head_rows_kernel<float>), grid, dim3(256), 0, st(stream), *a);
  return launched();
}

int dv_mix_gated_group_norm(int dtype, const float* y, int64_t ldy, const void* z, int64_t ldz, int64_t rows, int dim,
                            int groups, int padded, const float* w, float eps, void* out, void* stream) {
  if (!dtype_ok(dtype) || !y || !z || !w || !out || rows < 1 || dim < 1 || groups < 1 || dim % groups || padded < dim)
    return DV_ERR_INVALID_ARG;
  if (padded % 8 || ldy % 4 || ldz % 8 || !al16(y) || !al16(z) || !al16(w) || !al16(out)) return DV_ERR_ALIGNMENT;
  if (rows * groups >= (int64_t)1 << 31) return DV_ERR_UNSUPPORTED;
  const int gs = dim / groups;
#define DV_GROUP(T, W, VEC)                                                                                          \
  hipLaunchKernelGGL((gated_group_norm_kernel<T, W, VEC>), dim3(blocks_of(rows * groups, 4 / W)), dim3(256), 0, st(stream), \
                     y, ldy, (const T*)z, ldz, rows, dim, gs, padded, w, eps, (T*)out)
#define DV_GROUPS(T)                                  \
  do {                                                \
    if (gs % 4) DV_GROUP(T, 1, false);                \
    else if (gs <= 1024) DV_GROUP(T, 1, true);        \
    else DV_GROUP(T, 4, true);                        \
  } while (0)
  if (dtype == DV_BF16) DV_GROUPS(bf16_t);
  else DV_GROUPS(float);
#undef DV_GROUPS
#undef DV_GROUP
  return launched();
}

int dv_mix_rms_rows(int dtype, const void* x, int64_t ldx, int64_t rows, int dim, int padded, const float* w, float eps,
                    void* y, int64_t ldy, void* stream) {
  if (!dtype_ok(dtype) || !x || !w || !y || rows < 1 || dim < 1 || padded < dim) return DV_ERR_INVALID_ARG;
  if (padded % 8 || ldx % 8 || ldy % 8 || !al16(x) || !al16(y)) return DV_ERR_ALIGNMENT;
  const dim3 grid(blocks_of(rows, 4));
  if (dtype == DV_BF16)
    hipLaunchKernelGGL((rms_rows_kernel<bf16_t>), grid, dim3(256), 0, st(stream), (const bf16_t*)x, ldx, rows, dim, padded, w, eps, (bf16_t*)y, ldy);
  else
    hipLaunchKernelGGL((rms_rows_kernel<float>), grid, dim3(256), 0, st(stream), (const float*)x, ldx, rows, dim, padded, w, eps, (float*)y, ldy);
  return launched();
}

int dv_mix_gated_head_norm(int dtype, const float* o, const void* gate, int64_t ldg, int64_t rows, int heads, int vdim,
                           int padded, const float* w, float eps, void* y, void* stream) {
  if (!dtype_ok(dtype) || !o || !gate || !w || !y || rows < 1 || heads < 1 || vdim < 1 || padded < vdim)
    return DV_ERR_INVALID_ARG;
  if (padded % 8 || ldg % 8 || !al16(o) || !al16(gate) || !al16(y)) return DV_ERR_ALIGNMENT;
  const dim3 grid(blocks_of(rows * heads, 16));
  if (dtype == DV_BF16)
    hipLaunchKernelGGL((gated_head_norm_kernel<bf16_t>), grid, dim3(256), 0, st(stream), o, (const bf16_t*)gate, ldg, rows, heads, vdim, padded, w, eps, (bf16_t*)y);
  else
    hipLaunchKernelGGL((gated_head_norm_kernel<float>), grid, dim3(256), 0, st(stream), o, (const float*)gate, ldg, rows, heads, vdim, padded, w, eps, (float*)y);
  return launched();
}

int dv_mix_linear_row(int dtype, int before, int after, const dvRowArgs* a, void* stream) {
  if (!dtype_ok(dtype) || !a || !a->x || !a->W || a->M < 1 || a->K < 8) return DV_ERR_INVALID_ARG;
  if (a->K % 8 || a->ldw % 8 || !al16(a->W) || !al16(a->x)) return DV_ERR_ALIGNMENT;
  if (after != DV_OUT_RESIDUAL && after != DV_OUT_HYPER && !a->out) return DV_ERR_INVALID_ARG;
  if (after == DV_OUT_GLU && a->M % 2) return DV_ERR_INVALID_ARG;
  if (after == DV_OUT_RESIDUAL && (!a->res.x || !a->res.post.w || (a->res.h && !a->res.pre.w))) return DV_ERR_INVALID_ARG;
  if (after == DV_OUT_CONV && (!a->conv_w || a->taps < 1 || (a->taps > 1 && !a->conv_state) || a->conv_rows > a->M))
    return DV_ERR_INVALID_ARG;
  if (before == DV_ROW_RMS && (!a->xw || a->norm_dim < 1 || a->norm_dim > a->K)) return DV_ERR_INVALID_ARG;
  if (before == DV_ROW_HEADS && (!a->xw || !a->gate || a->head_stride < 8 || a->head_stride % 8 ||
                                 a->K % a->head_stride ||
                                 a->norm_dim < 1 || a->norm_dim > a->head_stride))
    return DV_ERR_INVALID_ARG;
  if (before == DV_ROW_GROUPS && (!a->xw || a->x_dim < 1 || a->x_dim > a->K || a->norm_dim < 1 || a->x_dim % a->norm_dim))
    return DV_ERR_INVALID_ARG;
  if ((before == DV_ROW_RMS || before == DV_ROW_GROUPS) && !al16(a->xw)) return DV_ERR_ALIGNMENT;
  if (after == DV_OUT_HYPER && (!a->hyper.x || !a->hyper.mix || !a->hyper.out || (a->hyper.u && !a->hyper.in) ||
                                a->hyper.streams < 1 || a->hyper.streams > DV_HYPER_ROW_MAX || a->hyper.width != a->M))
    return DV_ERR_INVALID_ARG;
  if (after == DV_OUT_GLU && a->bias) return DV_ERR_INVALID_ARG;
  if (a->side_x && (!a->side_w || !a->side_out || a->side_dim < 1)) return DV_ERR_INVALID_ARG;
  return dtype == DV_BF16 ? linear_row_any<bf16_t>(before, after, *a, st(stream))
                          : linear_row_any<float>(before, after, *a, st(stream));
}

int dv_mix_linear_tiles(int after, const dvTileArgs* a, void* stream) {
  if (!a || !a->x || !a->W || a->n < 1 || a->M < 1 || a->K < 8) return DV_ERR_INVALID_ARG;
  if (a->K % 8 || a->ldw % 8 || a->ldx % 8 || !al16(a->W) || !al16(a->x)) return DV_ERR_ALIGNMENT;
  if (after != DV_OUT_RESIDUAL && !a->out) return DV_ERR_INVALID_ARG;
  if (after == DV_OUT_GLU && a->M % 2) return DV_ERR_INVALID_ARG;
  if (after == DV_OUT_RESIDUAL && (!a->res.x || !a->res.post.w || (a->res.h && !a->res.pre.w))) return DV_ERR_INVALID_ARG;
  const int nt = a->n <= 16 ? 1 : (a->n <= 32 ? 2 : 4);
  const dim3 grid((a->M + 31) / 32, (a->n + 16 * nt - 1) / (16 * nt));
  if (grid.y > 65535) return DV_ERR_UNSUPPORTED;
#define DV_TILE(AFTER)                                                                                              \
  do {                                                                                                              \
    if (nt == 1) hipLaunchKernelGGL((linear_tiles_kernel<AFTER, 1>), grid, dim3(256), 0, st(stream), *a);            \
    else if (nt == 2) hipLaunchKernelGGL((linear_tiles_kernel<AFTER, 2>), grid, dim3(256), 0, st(stream), *a);       \
    else hipLaunchKernelGGL((linear_tiles_kernel<AFTER, 4>), grid, dim3(256), 0, st(stream), *a);                    \
  } while (0)
  switch (after) {
    case DV_OUT_F32: DV_TILE(DV_OUT_F32); break;
    case DV_OUT_T: DV_TILE(DV_OUT_T); break;
    case DV_OUT_GLU: DV_TILE(DV_OUT_GLU); break;
    case DV_OUT_RESIDUAL: DV_TILE(DV_OUT_RESIDUAL); break;
    default: return DV_ERR_UNSUPPORTED;
  }
#undef DV_TILE
  return launched();
}

int dv_mix_short_conv(int dtype, int out_f32, const dvConvArgs* a, void* stream) {
  if (!dtype_ok(dtype) || !a || !a->in || a->n < 1 || a->taps < 1 || !a->w || (a->taps > 1 && !a->state))
    return DV_ERR_INVALID_ARG;
  int heads = 0, widest = 0;
  for (const dvConvGroup& g : a->g) {
    if (g.heads < 0 || (g.heads > 0 && (!g.out || g.stride < 1 || g.dim < 1))) return DV_ERR_INVALID_ARG;
    heads += g.heads;
    if (g.heads > 0 && g.stride > widest) widest = g.stride;
  }
  if (heads == 0) return DV_ERR_INVALID_ARG;
  for (const dvConvGroup& g : a->g)
    if (g.heads > 0 && (g.stride % 8 || g.ld % 8 || !al16(g.out))) return DV_ERR_ALIGNMENT;
  if (a->ldi % 8 || !al16(a->in)) return DV_ERR_ALIGNMENT;
  if (dtype == DV_F32) return short_conv_types<float, float>(*a, heads, widest, st(stream));
  if (out_f32) return short_conv_types<bf16_t, float>(*a, heads, widest, st(stream));
  return short_conv_types<bf16_t, bf16_t>(*a, heads, widest, st(stream));
}

int dv_mix_conv_state(int dtype, const void* in, int64_t ldi, int n, int channels, int taps, float* state, void* stream) {
  if (!dtype_ok(dtype) || !in || n < 1 || channels < 1 || taps < 1 || (taps > 1 && !state)) return DV_ERR_INVALID_ARG;
  if (taps == 1) return DV_OK;
  const dim3 grid(blocks_of(channels, 256));
  if (dtype == DV_BF16)
    hipLaunchKernelGGL((conv_state_kernel<bf16_t>), grid, dim3(256), 0, st(stream), (const bf16_t*)in, ldi, n, channels, taps, state);
  else
    hipLaunchKernelGGL((conv_state_kernel<float>), grid, dim3(256), 0, st(stream), (const float*)in, ldi, n, channels, taps, state);
  return launched();
}

int dv_mix_ring_copy(int dtype, void* buf, int64_t ldb, void* ring, int cap, int64_t ldr, int first, int count, int width,
                     int to_ring, void* stream) {
  if (!dtype_ok(dtype) || !buf || !ring || cap < 1 || first < 0 || count < 0 || count > cap || width < 8)
    return DV_ERR_INVALID_ARG;
  if (width % 8 || ldb % 8 || ldr % 8 || !al16(buf) || !al16(ring)) return DV_ERR_ALIGNMENT;
  if (count == 0) return DV_OK;
  unsigned grid = blocks_of((int64_t)count * (width / 8), 256);
  if (grid > 4096) grid = 4096;
  if (dtype == DV_BF16)
    hipLaunchKernelGGL((ring_copy_kernel<bf16_t>), dim3(grid), dim3(256), 0, st(stream), (bf16_t*)buf, ldb, (bf16_t*)ring, cap, ldr, first, count, width, to_ring);
  else
    hipLaunchKernelGGL((ring_copy_kernel<float>), dim3(grid), dim3(256), 0, st(stream), (float*)buf, ldb, (float*)ring, cap, ldr, first, count, width, to_ring);
  return launched();
}

int dv_mix_attn_rows(int dtype, int q_f32, const dvAttnArgs* a, void* stream) {
  if (!dtype_ok(dtype)) return DV_ERR_INVALID_ARG;
  int rc = attn_args_ok(a);
  if (rc != DV_OK) return rc;
  if (!a->out) return DV_ERR_INVALID_ARG;
  if (dtype == DV_F32) rc = attn_rows_any<float, float>(*a, st(stream));
  else if (q_f32) rc = attn_rows_any<bf16_t, float>(*a, st(stream));
  else rc = attn_rows_any<bf16_t, bf16_t>(*a, st(stream));
  if (rc != DV_OK || a->splits == 1) return rc;
  const dim3 grid(a->H, (a->vdim_s + 63) / 64, a->n);
  if (dtype == DV_F32) hipLaunchKernelGGL((attn_merge_kernel<float, float>), grid, dim3(256), 0, st(stream), *a, (float*)a->out);
  else if (q_f32) hipLaunchKernelGGL((attn_merge_kernel<bf16_t, float>), grid, dim3(256), 0, st(stream), *a, (bf16_t*)a->out);
  else hipLaunchKernelGGL((attn_merge_kernel<bf16_t, bf16_t>), grid, dim3(256), 0, st(stream), *a, (bf16_t*)a->out);
  return launched();
}

int dv_mix_attn_tiles(const dvAttnArgs* a, int keys, void* stream) {
  int rc = attn_args_ok(a);
  if (rc != DV_OK) return rc;
  if (!a->out || a->ring > 0 || a->fresh_k || a->norm_dim > 0 || a->pos_dev || keys < 1 ||
      a->pos_host - a->base < 0 || a->pos_host - a->base + a->n > keys)
    return DV_ERR_INVALID_ARG;
  if (a->ldq % 8) return DV_ERR_ALIGNMENT;
  const int dt = (a->dim_s + 15) / 16, vt = (a->vdim_s + 31) / 32;
#define DV_TILES_V(DT)                                                        \
  do {                                                                        \
    if (vt <= 2) return attn_tiles_launch<DT, 2>(*a, keys, st(stream));       \
    if (vt <= 4) return attn_tiles_launch<DT, 4>(*a, keys, st(stream));       \
    if (vt <= 8) return attn_tiles_launch<DT, 8>(*a, keys, st(stream));       \
    return DV_ERR_UNSUPPORTED;                                                \
  } while (0)
  if (dt <= 4) DV_TILES_V(4);
  if (dt <= 8) DV_TILES_V(8);
  if (dt <= 12) DV_TILES_V(12);
  if (dt <= 16) DV_TILES_V(16);
#undef DV_TILES_V
  return DV_ERR_UNSUPPORTED;
}

int dv_mix_latent_absorb(int dtype, const float* q, const void* W, int H, int dim_s, int rank, float* out, void* stream) {
  if (!dtype_ok(dtype) || !q || !W || !out || H < 1 || dim_s < 1 || rank < 8) return DV_ERR_INVALID_ARG;
  if (rank % 8 || !al16(W)) return DV_ERR_ALIGNMENT;
  const dim3 grid(H, (rank + 127) / 128);
  if (dtype == DV_BF16)
    hipLaunchKernelGGL((latent_absorb_kernel<bf16_t>), grid, dim3(256), 0, st(stream), q, (const bf16_t*)W, dim_s, rank, out);
  else
    hipLaunchKernelGGL((latent_absorb_kernel<float>), grid, dim3(256), 0, st(stream), q, (const float*)W, dim_s, rank, out);
  return launched();
}

int dv_mix_latent_attn(int dtype, const dvAttnArgs* a, const void* W, int vrows, void* out, void* stream) {
  if (!dtype_ok(dtype) || !W || !out || vrows < 1 || !a || a->n != 1 || a->G != 1 || !a->part || a->splits < 2 ||
      a->k != a->v || a->dim_s != a->vdim_s || a->window > 0 || a->ring > 0 || a->base != 0 || a->fresh_k || a->norm_dim > 0)
    return DV_ERR_INVALID_ARG;
  int rc = attn_args_ok(a);
  if (rc != DV_OK) return rc;
  if (!al16(W) || !al16(a->part)) return DV_ERR_ALIGNMENT;
  const int rank = a->vdim_s;
  if (dtype == DV_F32) rc = attn_rows_any<float, float>(*a, st(stream));
  else if (rank <= 64) rc = latent_tiles<4>(*a, st(stream));
  else if (rank <= 128) rc = latent_tiles<8>(*a, st(stream));
  else if (rank <= 256) rc = latent_tiles<16>(*a, st(stream));
  else if (rank <= 512) rc = latent_tiles<32>(*a, st(stream));
  else rc = attn_rows_any<bf16_t, float>(*a, st(stream));
  if (rc != DV_OK) return rc;
  const dim3 grid(a->H, vrows <= 32 ? 1 : (vrows <= 64 ? 2 : 4));
  const size_t lds = (size_t)(rank / 4 < 256 ? 256 / (rank / 4) : 1) * rank * 4;
  if (dtype == DV_BF16)
    hipLaunchKernelGGL((latent_out_kernel<bf16_t>), grid, dim3(256), lds, st(stream), *a, (const bf16_t*)W, vrows, (bf16_t*)out);
  else
    hipLaunchKernelGGL((latent_out_kernel<float>), grid, dim3(256), lds, st(stream), *a, (const float*)W, vrows, (float*)out);
  return launched();
}

int dv_mix_delta_gates(int dtype, const void* z, int64_t ldz, const void* b, int64_t ldb, const float* A_log,
                       const float* dt_bias, int n, int heads, int dim_s, float* g, float* beta, void* stream) {
  if (!dtype_ok(dtype) || !z || !b || !A_log || !dt_bias || n < 1 || heads < 1 || dim_s < 1 || !g || !beta)
    return DV_ERR_INVALID_ARG;
  if (dim_s % 8 || ldz % 8 || !al16(z) || !al16(g) || !al16(dt_bias)) return DV_ERR_ALIGNMENT;
  const dim3 grid(blocks_of((int64_t)n * heads * dim_s / 4, 256));
  if (dtype == DV_BF16)
    hipLaunchKernelGGL((delta_gates_kernel<bf16_t>), grid, dim3(256), 0, st(stream), (const bf16_t*)z, ldz, (const bf16_t*)b, ldb, A_log, dt_bias, n, heads, dim_s, g, beta);
  else
    hipLaunchKernelGGL((delta_gates_kernel<float>), grid, dim3(256), 0, st(stream), (const float*)z, ldz, (const float*)b, ldb, A_log, dt_bias, n, heads, dim_s, g, beta);
  return launched();
}

int dv_mix_delta_scan(const dvDeltaArgs* a, void* stream) {
  if (!a || !a->q || !a->k || !a->v || !a->g || !a->beta || !a->S || !a->o || !a->tm || a->n < 1 || a->heads < 1 ||
      a->kv_heads < 1 || a->heads % a->kv_heads || a->dim_s < 8 || a->vdim_s < 1)
    return DV_ERR_INVALID_ARG;
  if (a->dim_s % 8 || !al16(a->q) || !al16(a->k) || !al16(a->g) || !al16(a->S) || !al16(a->tm)) return DV_ERR_ALIGNMENT;
  if (a->dim_s <= 64) return delta_scan<1>(*a, st(stream));
  if (a->dim_s <= 128) return delta_scan<2>(*a, st(stream));
  if (a->dim_s <= 192) return delta_scan<3>(*a, st(stream));
  if (a->dim_s <= 256) return delta_scan<4>(*a, st(stream));
  return DV_ERR_UNSUPPORTED;
}

int dv_mix_delta_step(int dtype, const dvDeltaStepArgs* a, void* stream) {
  if (!dtype_ok(dtype) || !a || !a->p || !a->Wa || !a->Wg || !a->A_log || !a->dt_bias || !a->S || !a->o || !a->gate ||
      a->heads < 1 || a->kv_heads < 1 || a->heads % a->kv_heads || a->dim < 1 || a->dim_s < a->dim || a->vdim_s < 1 ||
      a->rank_a < 8 || a->rank_g < 8)
    return DV_ERR_INVALID_ARG;
  if (a->dim_s % 8 || a->rank_a % 8 || a->rank_g % 8 || !al16(a->Wa) || !al16(a->Wg) || !al16(a->S)) return DV_ERR_ALIGNMENT;
  const dim3 grid((unsigned)(a->heads * ((a->vdim_s + kDeltaCols - 1) / kDeltaCols)));
  const size_t lds = (size_t)(a->rank_a + a->rank_g) * 4;
  if (lds > 40 * 1024) return DV_ERR_UNSUPPORTED;
#define DV_STEP(T)                                                                                                  \
  do {                                                                                                              \
    if (a->dim_s <= 64) hipLaunchKernelGGL((delta_decode_kernel<T, 4>), grid, dim3(256), lds, st(stream), *a);       \
    else if (a->dim_s <= 128) hipLaunchKernelGGL((delta_decode_kernel<T, 8>), grid, dim3(256), lds, st(stream), *a); \
    else if (a->dim_s <= 192) hipLaunchKernelGGL((delta_decode_kernel<T, 12>), grid, dim3(256), lds, st(stream), *a); \
    else if (a->dim_s <= 256) hipLaunchKernelGGL((delta_decode_kernel<T, 16>), grid, dim3(256), lds, st(stream), *a); \
    else return DV_ERR_UNSUPPORTED;                                                                                 \
  } while (0)
  if (dtype == DV_BF16) DV_STEP(bf16_t);
  else DV_STEP(float);
#undef DV_STEP
  return launched();
}

int dv_mix_ssd_scan(int dtype, const dvSsdArgs* a, void* stream) {
  if (!dtype_ok(dtype) || !a || !a->xbc || !a->dt || !a->A_log || !a->dt_bias || !a->D || !a->S || !a->y || !a->tm || a->n < 1 ||
      a->heads < 1 || a->groups < 1 || a->heads % a->groups || a->vdim < 1 || a->state_s < 8)
    return DV_ERR_INVALID_ARG;
  if (a->state_s % 8 || a->ld % 4 || a->off_b % 4 || a->off_c % 4 || !al16(a->xbc) || !al16(a->S) || !al16(a->tm))
    return DV_ERR_ALIGNMENT;
  return dtype == DV_BF16 ? ssd_scan_any<bf16_t>(*a, st(stream)) : ssd_scan_any<float>(*a, st(stream));
}

int dv_mix_ssd_step(const dvSsdStepArgs* a, void* stream) {
  if (!a || !a->p || !a->A_log || !a->dt_bias || !a->D || !a->S || !a->y || a->heads < 1 || a->groups < 1 ||
      a->heads % a->groups || a->vdim < 1 || a->state_s < 8)
    return DV_ERR_INVALID_ARG;
  if (a->state_s % 8 || a->off_b % 4 || a->off_c % 4 || !al16(a->p) || !al16(a->S)) return DV_ERR_ALIGNMENT;
  const dim3 grid((unsigned)(a->heads * ((a->vdim + kSsdCols - 1) / kSsdCols)));
  if (a->state_s <= 64) hipLaunchKernelGGL((ssd_step_kernel<1>), grid, dim3(256), 0, st(stream), *a);
  else if (a->state_s <= 128) hipLaunchKernelGGL((ssd_step_kernel<2>), grid, dim3(256), 0, st(stream), *a);
  else if (a->state_s <= 192) hipLaunchKernelGGL((ssd_step_kernel<3>), grid, dim3(256), 0, st(stream), *a);
  else if (a->state_s <= 256) hipLaunchKernelGGL((ssd_step_kernel<4>), grid, dim3(256), 0, st(stream), *a);
  else return DV_ERR_UNSUPPORTED;
  return launched();
}

int dv_mix_greedy_advance(const float* logits, int vocab, void* token, void* position, void* seq_pos, void* sequences,
                          int64_t seq_capacity, void* out_index, float* scores, int64_t score_ld, int64_t score_rows,
                          void* score_index, void* stream) {
  if (!logits || vocab < 1 || !token || !position || !seq_pos || !sequences || !out_index || seq_capacity < 0 ||
      (scores && (!score_index || score_ld < vocab || score_rows < 0)))
    return DV_ERR_INVALID_ARG;
  hipLaunchKernelGGL(greedy_advance_f32_kernel, dim3(1), dim3(1024), 0, st(stream), logits, vocab, (int64_t*)token,
                     (int64_t*)position, (int*)seq_pos, (int64_t*)sequences, (int64_t*)out_index, scores, score_ld,
                     (int64_t*)score_index, seq_capacity, score_rows);
  return launched();
}

}  // extern "C"
