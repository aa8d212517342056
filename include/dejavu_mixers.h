/*
 * C ABI of libdejavu_mixers.so: gfx950 kernels for decoders that mix tokens with latent attention, a gated delta
 * rule, a Mamba-2 recurrence, or sliding-window or chunk-local attention, around dynamic-tanh norms and one residual
 * stream or around RMS norms and several streams (see dejavu_amd/mixers.py for the modules).
 *
 * Conventions
 *  - every pointer is a DEVICE pointer; the structs themselves live on the host and are copied by the call;
 *  - `dtype` selects the element type of weights and activations: DV_BF16 or DV_F32.  Sums, norms, scores, the
 *    residual stream and the recurrent state are fp32 either way;
 *  - sizes along a vectorised dimension (columns of a weight, channels of a head) are multiples of 8; what a model
 *    lacks is zero padding in weights and activations.  Rows start on 16-byte boundaries;
 *  - calls only enqueue work on `stream` (a hipStream_t): no allocation, no synchronisation;
 *  - return value: DV_OK or a negative DV_ERR_* code (dejavu_hip.h).
 */
#ifndef DEJAVU_MIXERS_H
#define DEJAVU_MIXERS_H

#include "dejavu_hip.h"

#ifdef __cplusplus
extern "C" {
#endif

#define DV_BF16 0
#define DV_F32 1

/* Dynamic tanh: tanh(alpha x) w + b, per channel. */
typedef struct {
  const float* w;
  const float* b;
  float alpha;
} dvDynTanh;

/* What follows a sublayer's last product: x += post(y); x += x0 (x0 non-null); h = pre(x) (h non-null). */
typedef struct {
  float* x;
  const float* x0;
  void* h;
  dvDynTanh post, pre;
} dvResidual;

/* Several residual streams x [n][streams][width] around a sublayer with result y:
 * x_t <- sum_s mix[s][t] x_s + out[t] y, all at once; then u = sum_t in[t] x_t for the next sublayer (in null: none). */
#define DV_HYPER_MAX 16        /* streams                                                    */
#define DV_HYPER_ROW_MAX 4     /* streams in the epilogue of dv_mix_linear_row               */
typedef struct {
  float* x;
  const float* mix;        /* [streams][streams], from, to */
  const float* out;        /* [streams] */
  const float* in;         /* [streams] */
  float* u;                /* [n][width] or null */
  int streams, width;
} dvHyper;

/* An RMS norm that follows: h = u / rms(u) * w, the mean over dim entries, eps inside the root (h null: none). */
typedef struct {
  const float* w;
  float eps;
  int dim;
  void* h;
} dvRmsOut;

/* Gated units of a feed-forward. */
#define DV_GLU_CLAMPED 0   /* g = min(gate, limit), u = clamp(up, limit): g sigmoid(1.702 g) (u + 1) */
#define DV_GLU_RELU 1      /* max(gate, 0) up                                                         */

/* How a row enters dv_mix_linear_row, and what happens to the products. */
#define DV_ROW_PLAIN 0   /* x: elements of `dtype`                                                        */
#define DV_ROW_RMS 1     /* x: fp32, divided by its root mean square over norm_dim, times xw              */
#define DV_ROW_HEADS 2   /* x: fp32 heads of head_stride entries, each RMS-normed, times xw, times gate   */
#define DV_ROW_GROUPS 3  /* x: fp32, groups of norm_dim entries (x_dim in all) each RMS-normed, times xw  */
#define DV_OUT_F32 0     /* fp32 store                                                                    */
#define DV_OUT_T 1       /* store in `dtype`                                                              */
#define DV_OUT_GLU 2     /* rows 2 i (gate) and 2 i + 1 (up) -> gated unit `act`, in `dtype`               */
#define DV_OUT_RESIDUAL 3 /* dvResidual                                                                   */
#define DV_OUT_CONV 4    /* fp32; the first conv_rows rows pass a short convolution (and silu)            */
#define DV_OUT_HYPER 5   /* dvHyper, at most DV_HYPER_ROW_MAX streams                                     */

typedef struct {
  const void* x;
  const void* W;           /* [M][ldw] */
  int64_t ldw;
  int M, K;
  const float* xw;
  const float* gate;       /* [K] factors of DV_ROW_HEADS */
  float eps;
  int norm_dim, head_stride, x_dim;
  const void* bias;        /* [M] in `dtype` or null; added to the products (not with DV_OUT_GLU) */
  void* out;
  int act;
  float limit;
  dvResidual res;
  dvHyper hyper;
  const float* conv_w;     /* [conv_rows][taps] */
  const float* conv_b;     /* [conv_rows] or null */
  float* conv_state;       /* [conv_rows][taps - 1], oldest first, moved on by one token */
  int conv_rows, taps, silu;
  /* a second fp32 row that one extra workgroup RMS-norms and stores at row `position` of side_out (null: none) */
  const float* side_x;
  const float* side_w;
  void* side_out;
  int64_t side_ld;
  int side_dim, side_padded;
  const int* pos_dev;      /* position: *pos_dev, or pos_host when null */
  int pos_host;
} dvRowArgs;

/* Products of a few rows on the matrix cores, bf16: out [n][M] = x [n][K] W^T. */
typedef struct {
  const void* x;
  int64_t ldx;
  const void* W;
  int64_t ldw;
  int n, M, K;
  const void* bias;        /* [M] or null (not with DV_OUT_GLU) */
  void* out;               /* DV_OUT_F32 / DV_OUT_T: [n][ldo]; DV_OUT_GLU: [n][ldo], M / 2 columns */
  int64_t ldo;
  int act;
  float limit;
  dvResidual res;          /* DV_OUT_RESIDUAL: x, x0, h are [n][M] */
} dvTileArgs;

/* One group of heads of a short convolution's output. */
typedef struct {
  int heads, stride, dim;  /* channels per head: stride in memory, dim real ones */
  int norm;                /* 0: none; 1: / root mean square over dim; 2: unit vector, times scale */
  float eps, scale;
  void* out;               /* [n][heads][stride], ld elements between tokens */
  int64_t ld;
} dvConvGroup;
typedef struct {
  const void* in;          /* [n][ldi], the groups' channels one after the other */
  int64_t ldi;
  int n, taps, silu;
  const float* w;          /* [channels][taps] */
  const float* b;          /* [channels] or null */
  const float* state;      /* [channels][taps - 1] */
  dvConvGroup g[3];
} dvConvArgs;

/* One group of heads of a projection's rows: RMS-normed per head with a weight, or mixed with other rows. */
typedef struct {
  int heads, stride, dim;
  const float* w;          /* [stride]: x / rms(x) * w, the mean over dim; null: no norm */
  float eps;
  const void* other;       /* no norm: (1 - *lambda) x + *lambda other (null: x) */
  int64_t ldo;
  const float* lambda;
  void* out;               /* [n][heads][stride], ld elements between tokens */
  int64_t ld;
} dvHeadGroup;
typedef struct {
  const void* in;          /* [n][ldi], the groups' channels one after the other */
  int64_t ldi;
  int n;
  dvHeadGroup g[3];
} dvHeadArgs;

/* Softmax attention of n query rows; scores (q . k) * scale, fp32. */
typedef struct {
  const void* q;
  int64_t ldq;
  const void* k;
  int64_t ldk, k_head;
  const void* v;
  int64_t ldv, v_head;
  int n, H, G, dim_s, vdim_s;
  float scale;
  const float* sink;       /* [H] or null: exp(sink) joins the denominator */
  const void* gate;        /* [n][ldg] logits or null: outputs times sigmoid(gate[., head]) */
  int64_t ldg;
  int window;              /* > 0: a query sees the newest `window` tokens up to itself */
  int chunk;               /* > 0 (without a window): a query sees the tokens of its own chunk up to itself; chunks
                            * are counted from position 0 */
  const float* rel;        /* [H][rel_len] or null: added to the scaled score by distance, the last entry beyond */
  int rel_len;
  int ring;                /* > 0: token j lies in row j % ring of k and v, else in row j - base */
  int base;
  const int* pos_dev;      /* position of query row 0 */
  int pos_host;
  void* out;               /* [n][H][vdim_s] */
  float* part;             /* splits > 1 (at most 128): n H splits (vdim_s + 2) floats of scratch */
  int splits;
  const float* fresh_k;    /* decode: this token's key / value rows (fp32), stored in their slots first */
  const float* fresh_v;
  int norm_dim;            /* > 0: q and fresh_k are divided by their root mean square over norm_dim */
  float eps;
  const float* q_w;        /* [dim_s] or null: weights of these norms */
  const float* k_w;
  const float* other_v;    /* fp32 [G][vdim_s] or null: fresh_v <- (1 - *lambda) fresh_v + *lambda other_v */
  const float* lambda;
} dvAttnArgs;

typedef struct {
  const float* q;          /* [n][kv_heads][dim_s] */
  const float* k;
  const float* v;          /* [n][heads][vdim_s] */
  const float* g;          /* [n][heads][dim_s] decays */
  const float* beta;       /* [n][heads] */
  float* S;                /* [heads][vdim_s][dim_s] */
  float* o;                /* [n][heads][vdim_s] */
  float* tm;               /* scratch of tm_floats: ceil(min(n, 4096) / 16) * heads * (49 D + 512), */
  int64_t tm_floats;       /* D: dim_s rounded up to a multiple of 64 */
  int n, heads, kv_heads, dim_s, vdim_s;
} dvDeltaArgs;

/* One decode token of the gated delta rule from the fp32 projection row p. */
typedef struct {
  const float* p;          /* q, k, v after convolution and silu; then the rows at off_b, off_a, off_g */
  int off_k, off_v, off_b, off_a, off_g;
  int heads, kv_heads, dim, dim_s, vdim_s;
  const void* Wa;          /* [heads * dim_s][rank_a] */
  const void* Wg;          /* [heads * vdim_s][rank_g] */
  int rank_a, rank_g;
  const float* A_log;
  const float* dt_bias;
  float* S;
  float* o;                /* [heads][vdim_s] */
  float* gate;             /* [heads][vdim_s]: sigmoid of the output gate */
} dvDeltaStepArgs;

/* Mamba-2 recurrence over n tokens: S <- exp(-exp(A_log) dt) S + dt B x^T, y = S^T C + D x per head, where
 * dt = softplus(logit + dt_bias); head h uses group h / (heads / groups) of B and C. */
typedef struct {
  const float* xbc;        /* [n][ld]: x [heads][vdim], then from off_b on B and from off_c on C, [groups][state_s];
                            * rows n .. up to the next multiple of 64 are readable and finite */
  int64_t ld;
  int off_b, off_c;
  const void* dt;          /* [n][lddt] logits in `dtype`, a column per head */
  int64_t lddt;
  const float* A_log;      /* [heads] each */
  const float* dt_bias;
  const float* D;
  float* S;                /* [heads][vdim][state_s] */
  float* y;                /* [n][ldy], [heads][vdim] */
  int64_t ldy;
  float* tm;               /* scratch of tm_floats: ceil(min(n, 4096) / 64) * heads * 2688 */
  int64_t tm_floats;
  int n, heads, groups, vdim, state_s;
} dvSsdArgs;

/* One decode token of it from the fp32 projection row p (x, B, C after convolution and silu; z and dt logits);
 * y [heads][vdim] is also multiplied by silu(z). */
typedef struct {
  const float* p;
  int off_b, off_c, off_z, off_dt;
  const float* A_log;
  const float* dt_bias;
  const float* D;
  float* S;
  float* y;
  int heads, groups, vdim, state_s;
} dvSsdStepArgs;

/* Embedding of a token and its predecessor: embed[token] scale + bigram[row], row = (previous mul_prev + token
 * mul_cur) mod buckets, or `buckets` for the first token of a sequence; every stream starts with it. */
typedef struct {
  const void* tokens;      /* [n] int64 */
  void* history;           /* [capacity] int64: the sequence's tokens by position, written here */
  int64_t capacity, vocab;
  const void* embed;       /* [vocab][width] */
  float scale;
  const void* bigram;      /* [buckets + 1][width] or null */
  int64_t buckets, mul_prev, mul_cur;
  const int* pos_dev;
  int pos_host, n;
} dvEmbedArgs;

/* x = x0 = embed[token] (x0 may be null), h = norm(x). */
DV_API int dv_mix_embed(int dtype, const void* tokens, int64_t vocab, const void* embed, int n, int width, float* x,
                        float* x0, const dvDynTanh* norm, void* h, void* stream);
/* Residual step of n x width values y (null: only x += x0 and h = pre(x)). */
DV_API int dv_mix_residual(int dtype, const void* y, int64_t n, int width, const dvResidual* r, void* stream);
/* y [n][ff] from gu [n][2 ff] (gate and up interleaved): the gated unit `act` (DV_GLU_*). */
DV_API int dv_mix_glu(int dtype, const void* gu, int64_t count, int act, float limit, void* y, void* stream);
/* Streams: start of a portion (r->mix, r->out are not read). */
DV_API int dv_mix_hyper_embed(int dtype, const dvEmbedArgs* e, const dvHyper* r, const dvRmsOut* norm, void* stream);
/* Streams: what follows a sublayer with n x width values y (null: only u and h, the streams stay). */
DV_API int dv_mix_hyper_rows(int dtype, const void* y, int n, const dvHyper* r, const dvRmsOut* norm, void* stream);
DV_API int dv_mix_head_rows(int dtype, const dvHeadArgs* args, void* stream);
/* out = t / rms(t) * w per group of `dim / groups` entries, t = y silu(z); entries dim .. padded - 1 become 0. */
DV_API int dv_mix_gated_group_norm(int dtype, const float* y, int64_t ldy, const void* z, int64_t ldz, int64_t rows,
                                   int dim, int groups, int padded, const float* w, float eps, void* out, void* stream);
/* y = x / rms(x) * w, row by row; w has `padded` entries, the mean runs over `dim`. */
DV_API int dv_mix_rms_rows(int dtype, const void* x, int64_t ldx, int64_t rows, int dim, int padded, const float* w,
                           float eps, void* y, int64_t ldy, void* stream);
/* y = o / rms(o) * w * sigmoid(gate) per head; o fp32 [rows][heads][padded]. */
DV_API int dv_mix_gated_head_norm(int dtype, const float* o, const void* gate, int64_t ldg, int64_t rows, int heads,
                                  int vdim, int padded, const float* w, float eps, void* y, void* stream);
DV_API int dv_mix_linear_row(int dtype, int before, int after, const dvRowArgs* args, void* stream);
DV_API int dv_mix_linear_tiles(int after, const dvTileArgs* args, void* stream);
DV_API int dv_mix_short_conv(int dtype, int out_f32, const dvConvArgs* args, void* stream);
DV_API int dv_mix_conv_state(int dtype, const void* in, int64_t ldi, int n, int channels, int taps, float* state,
                             void* stream);
/* Rows of a portion's buffer <-> a ring of cap rows, token first .. first + count - 1 (count <= cap). */
DV_API int dv_mix_ring_copy(int dtype, void* buf, int64_t ldb, void* ring, int cap, int64_t ldr, int first, int count,
                            int width, int to_ring, void* stream);
/* q_f32: the queries (and gate logits) are fp32 instead of `dtype`. */
DV_API int dv_mix_attn_rows(int dtype, int q_f32, const dvAttnArgs* args, void* stream);
/* bf16, a portion on the matrix cores; `keys` rows behind k and v (contiguous, ring = 0). */
DV_API int dv_mix_attn_tiles(const dvAttnArgs* args, int keys, void* stream);
/* Latent decode row: out [H][rank] = q[h] W_uk[h]; W [H][dim_s][rank]. */
DV_API int dv_mix_latent_absorb(int dtype, const float* q, const void* W, int H, int dim_s, int rank, float* out,
                                void* stream);
/* Latent decode row: attention over the cache (args: G = 1, k == v, dim_s = vdim_s = rank, at least two splits with
 * `part`, q and gate fp32), gated, times W_uv [H][vrows][rank]; out [H][vrows]. */
DV_API int dv_mix_latent_attn(int dtype, const dvAttnArgs* args, const void* W, int vrows, void* out, void* stream);
DV_API int dv_mix_delta_gates(int dtype, const void* z, int64_t ldz, const void* b, int64_t ldb, const float* A_log,
                              const float* dt_bias, int n, int heads, int dim_s, float* g, float* beta, void* stream);
DV_API int dv_mix_delta_scan(const dvDeltaArgs* args, void* stream);
DV_API int dv_mix_delta_step(int dtype, const dvDeltaStepArgs* args, void* stream);
DV_API int dv_mix_ssd_scan(int dtype, const dvSsdArgs* args, void* stream);
DV_API int dv_mix_ssd_step(const dvSsdStepArgs* args, void* stream);
/* dv_greedy_advance_f16 for fp32 logits. */
DV_API int dv_mix_greedy_advance(const float* logits, int vocab, void* token, void* position, void* seq_pos,
                                 void* sequences, int64_t seq_capacity, void* out_index, float* scores,
                                 int64_t score_ld, int64_t score_rows, void* score_index, void* stream);

#ifdef __cplusplus
}
#endif
#endif
