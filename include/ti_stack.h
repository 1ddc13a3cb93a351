/*
 * ti_stack.h -- extern "C" kernels of the layer-stack models (models described layer by layer by
 * their config.json; ti_engine.h ti_engine_create_stack drives them).
 *
 * Two element types share every kernel: TI_DT_BF16 (bf16 weights, activations and cache, fp32
 * accumulation) and TI_DT_F32 (everything fp32; v_mfma_f32_16x16x4_f32 is true fp32).  The residual
 * stream, norms, router, rotary angles, attention scores and softmax are fp32 in both.
 *
 * Operand geometry: an MFMA operand fragment is 64 lanes x 16 bytes; lane l holds row (l & 15),
 * elements [VEC * (l >> 4), +VEC) of a k-tile of KT = 4 * VEC elements (bf16: VEC 8, KT 32; fp32:
 * VEC 4, KT 16).  Weights are stored fragment by fragment: [ceil(N / 16)][Kp / KT][64][VEC], Kp = K
 * rounded up to 128 bytes, zero padded.  Activations are row-major with a row pitch of >= Kp
 * elements whose padding is zero.
 */
#ifndef TI_STACK_H
#define TI_STACK_H

#include <stddef.h>
#include <stdint.h>

#include "ti_hip.h"

#ifdef __cplusplus
extern "C" {
#endif

enum ti_dtype { TI_DT_BF16 = 0, TI_DT_F32 = 1 };

/* K rounded up to whole 128-byte spans of `dtype` elements; N x K weight bytes in fragment order. */
int ti_stack_kpad(int dtype, int K);
size_t ti_stack_weight_bytes(int dtype, int N, int K);
/* Pack fp32 device elements src[r * row_stride + k * k_stride] (r < rows, k < K) into fragment order:
 * row r becomes destination row row_map[r] (device; NULL: r), which must lie inside dst; other
 * elements of dst are left as they are (zero padding is the allocation's). */
int ti_stack_pack(const float* src, int64_t row_stride, int64_t k_stride, int rows, int K, const int32_t* row_map,
                  int dtype, void* dst, ti_stream_t s);
/* n fp32 elements to `dtype` (embedding tables). */
int ti_stack_convert(const float* src, uint64_t n, int dtype, void* dst, ti_stream_t s);

/* ------------------------------------------------------------------- dense products */
enum ti_dense_epi {
  TI_DE_F32 = 0,     /* out fp32 [m][n] = v (+ add[n])                                       */
  TI_DE_T,           /* out T [m][n]                                                         */
  TI_DE_SWIGLU,      /* columns (2j, 2j + 1) = (gate, up): out T [m][j] = silu(gate) * up    */
  TI_DE_ROPE,        /* out T [m][n]; column n of head n / head_w, at r = n % head_w >= rot_off,
                        rotated in adjacent pairs by rope_cs[pos[m]][(r - rot_off) / 2]      */
  TI_DE_GATE,        /* out T [m][batch * N + n] = v * gate[m][batch]                        */
  TI_DE_LOGITS,      /* out fp32 + greedy argmax keys (ti_hip.h TI_EPI_LOGITS_ARGMAX)        */
  TI_DE_KFRAG,       /* rows are keys, columns (head, head_w): key fragments of every head,
                        out T [head][key / 16][head_w / KT][64][VEC]                         */
  TI_DE_VFRAG,       /* rows are keys, columns (head, head_w): transposed value fragments,
                        out T [head][head_w / 16][key / KT][64][VEC] (ti_latent_attn_prefill) */
  TI_DE_ACT,         /* v += add[n] (nullable); columns n < act_cols through `act`; columns n < t_cols
                        to out T [m][n], the others to out2 fp32 [m][n - t_cols]             */
  TI_DE_LRU          /* gates of a real-gated linear recurrent unit over a prompt chunk, one batch per
                        diagonal block: columns (2j, 2j + 1) = (recurrence, input) gate of the block's
                        channel j.  log a = -sigmoid(r) * lru_rate, b = sqrt(1 - a^2) * sigmoid(i) * u;
                        out fp32 [m][channel][2] = (a, b) (ti_lru_scan)                      */
};
enum ti_act { TI_ACT_NONE = 0, TI_ACT_GELU_TANH, TI_ACT_GELU_ERF };

typedef struct ti_dense_args {
  const void* w;               /* fragment-ordered weights                                   */
  int64_t w_batch;             /* elements between the weights of consecutive batches / experts */
  const void* a;               /* activations T, row-major                                   */
  int64_t a_batch;             /* elements between batches                                   */
  void* out;
  int64_t o_batch;
  int32_t lda, ldo;
  int32_t M, N, K;             /* K: the padded k extent (ti_stack_kpad)                     */
  int32_t batch;               /* independent products (heads); 1 otherwise                  */
  int32_t epi, dtype;
  const float* add;            /* TI_DE_F32, nullable                                        */
  const float* rope_cs;        /* TI_DE_ROPE: [position][(head_w - rot_off) / 2][2]          */
  const int32_t* pos;          /* [M]                                                        */
  int32_t head_w, rot_off;
  const float* gate;           /* TI_DE_GATE: [M][gate_ld]                                   */
  int32_t gate_ld;
  int32_t key_blocks;          /* TI_DE_KFRAG / VFRAG: 16-key blocks the output holds per head */
  unsigned long long* argmax;  /* TI_DE_LOGITS */
  int32_t* step_ctr;           /* TI_DE_LOGITS, nullable: += advance once                    */
  int32_t advance;
  /* grouped products (experts): tile t covers entries [first, first + rows) of expert e's list */
  int32_t tile_rows;           /* 0 = not grouped; 16, 64 or 128: rows a tile holds; 1: tile t is
                                  entry t alone, of expert tiles[t]                           */
  int32_t max_tiles;           /* tiles launched; those at or past *n_tiles return at once   */
  const int32_t* tiles;        /* device [max_tiles][4] = expert, first, rows, -             */
  const int32_t* n_tiles;      /* device                                                     */
  const int32_t* rows_in;      /* entry p reads activation row (rows_in ? rows_in[p] : p) / row_div */
  const int32_t* rows_out;     /* nullable: entry p writes output row rows_out[p]            */
  int32_t row_div;
  /* TI_DE_ACT */
  int32_t act, act_cols, t_cols, ld2;
  float* out2;
  /* TI_DE_LRU: batch b's columns are channels [b * N / 2, +N / 2); u is the product's own activation
   * row (element [m][b * a_batch + j] of `a`), add [batch * N] the gates' biases in column order */
  const float* lru_rate;       /* [channels] 8 * softplus(lambda)                            */
} ti_dense_args;
int ti_dense(const ti_dense_args* a, ti_stream_t s);
size_t ti_dense_args_bytes(void);

/* ------------------------------------------------------------------- norms and residual
 * One row per workgroup:
 *   y' = post_w ? norm(y; post_w, post_b) : y           (y: fp32 rows, or the weighted expert outputs
 *   x  = x + y'                                          sum_k part_w[m][k] * parts[m * top + k])
 *   xn = T(norm(x; w, b)) (w NULL: T(x))  and / or  cat = T([x ; x0])
 * Any of the three parts may be absent.  kind 0: layer norm (x - mean) / sqrt(var + eps) * w + b;
 * kind 1: RMS norm x / sqrt(mean(x^2) + eps) * w (b ignored). */
enum ti_norm_kind { TI_NORM_LAYER = 0, TI_NORM_RMS = 1 };
typedef struct ti_rownorm_args {
  float* x;                    /* residual [M][H] fp32, updated when y or parts is given     */
  const float* y;              /* nullable [M][ldy]                                          */
  const void* parts;           /* nullable T [M * top][ldy]                                  */
  const float* part_w;         /* [M][top]                                                   */
  const float* post_w;
  const float* post_b;
  const float* w;              /* nullable: xn without a norm                                */
  const float* b;
  void* xn;                    /* nullable T [M][ldn]                                        */
  const float* x0;             /* with cat: [M][H]                                           */
  void* cat;                   /* nullable T [M][ldc]: [x ; x0]                              */
  float eps;
  int32_t M, H, ldy, ldn, ldc, top, kind, dtype;
  /* nullable: also route the normalised row (ti_route's choice) with fragment-ordered router weights
   * [route_e][H], where ti_rownorm_routes(H, route_e) */
  const void* route_w;
  int32_t* route_idx;          /* [M][route_top] */
  float* route_wgt;
  int32_t route_e, route_top;
} ti_rownorm_args;
int ti_rownorm(const ti_rownorm_args* a, ti_stream_t s);
int ti_rownorm_routes(int H, int E);

/* ------------------------------------------------------------------- expert routing
 * logits fp32 [M][ld]: softmax over E experts, the `top` largest scores (lowest index first among
 * equals), not renormalised: idx [M][top], wgt [M][top].  Then the (row, expert) entries grouped by
 * expert: list[p] = row * top + k, and tiles of at most tile_rows entries of one expert.
 * E <= 1024, top <= min(E, 64).  tile_rows 0: idx / wgt only; logits NULL: grouping of a given idx only. */
typedef struct ti_route_args {
  const float* logits;
  int32_t ld, M, E, top;
  int32_t* idx;
  float* wgt;
  int32_t* list;               /* [M * top]                                                  */
  int32_t* tiles;              /* [ti_route_max_tiles][4]                                    */
  int32_t* n_tiles;
  int32_t tile_rows;
} ti_route_args;
int ti_route_max_tiles(int M, int E, int top, int tile_rows);
int ti_route(const ti_route_args* a, ti_stream_t s);

/* ------------------------------------------------------------------- latent attention
 * The cache row of a position is [latent (lat_p) | rotated key part (rot_p)] T, lat_p / rot_p the
 * latent and rotated sizes padded to KT elements; a slot holds seq_p rows (max_seq rounded up to 128).
 *
 * ti_latent_prep: per row, from the fused projection a32 [M][lda] fp32 (query latent at 0, latent at
 * lat_off, rotated part at rot_off (adjacent pairs), gate logits at gate_off):
 *   cq [M][ldq] T = rms_norm(query latent; q_w);  cache row pos[m] = [rms_norm(latent; c_w) | rotated];
 *   gate [M][heads] fp32 = sigmoid.  Row m's cache slot is cache + m * slot_stride. */
typedef struct ti_latent_prep_args {
  const float* a32;
  int32_t lda, M, q_rank, kv_rank, rot_dim, heads, lat_off, rot_off, gate_off;
  const float* q_w;
  const float* c_w;
  const float* rope_cs;        /* [position][rot_p / 2][2] */
  const int32_t* pos;
  void* cq;
  int32_t ldq;
  void* cache;
  int64_t slot_stride;         /* elements; 0: all rows share one slot (prompt chunk)        */
  int32_t lat_p, rot_p;
  float* gate;
  float eps;
  int32_t dtype;
  const int32_t* slot;         /* nullable [M]: stream slot of row m (NULL: m)               */
} ti_latent_prep_args;
int ti_latent_prep(const ti_latent_prep_args* a, ti_stream_t s);

/* Once per process and device, before a capture: lifts the LDS limit of the kernels below. */
int ti_latent_prepare(void);

/* Decode attention in latent space: scores (qa . latent + qr . rotated) * scale over keys
 * [0, pos[m]], softmax whose denominator also holds exp(sink[h]), out = weights . latents.
 * qa T [M][heads][lat_p] (the query carried through the key up-projection), qr T rows of `ldqr`
 * elements per (m, head) with the rotated part at qr_off.  out T [M][heads][lat_p].
 * splits > 1 (at most 64): part_o T [M][splits][heads][lat_p] and part_ml fp32 [M][splits][heads][2]
 * hold each split's normalised row and (max, sum); out non-NULL: a second launch merges them, NULL: left
 * to ti_latent_attn_out. */
typedef struct ti_latent_attn_args {
  const void* qa;
  const void* q;               /* T [M][heads][ldqr]; rotated part at qr_off                 */
  int32_t ldqr, qr_off;
  const void* cache;
  int64_t slot_stride;
  const int32_t* pos;
  const float* sink;
  float scale;
  void* out;
  void* part_o;
  float* part_ml;
  int32_t M, heads, lat_p, rot_p, splits, seq_p, dtype;
  const int32_t* slot;         /* nullable [M]: stream slot of row m (NULL: m)               */
} ti_latent_attn_args;
int ti_latent_attn_decode(const ti_latent_attn_args* a, ti_stream_t s);
/* Merge of the splits, value up-projection and head gate: out T [M][ldo], head h's vdim values at
 * h * vdim.  w: fragment-ordered, w_batch elements per head ([vdim][lat_p]). */
typedef struct ti_latent_out_args {
  const void* part_o;
  const float* part_ml;
  const float* sink;
  const void* w;
  int64_t w_batch;
  const float* gate;           /* [M][heads]                                                 */
  void* out;
  int32_t ldo, M, heads, lat_p, vdim, splits, dtype;
} ti_latent_out_args;
int ti_latent_attn_out(const ti_latent_out_args* a, ti_stream_t s);
int ti_latent_attn_splits(int M, int heads, int max_seq);

/* Prompt-chunk attention over keys and values expanded per head (TI_DE_KFRAG / TI_DE_VFRAG), rows
 * [0, M) of one slot at positions pos0 + m; out T [M][ldo] gets head h's vdim values at h * vdim,
 * times gate[m][h].  q T [M][heads][dim_p + rot_p]; the rotated key part is read from the cache. */
typedef struct ti_latent_prefill_args {
  const void* q;
  const void* kfrag;
  const void* vfrag;
  const void* cache;           /* the slot's rows                                            */
  const float* sink;
  const float* gate;           /* [M][heads]                                                 */
  void* out;
  float scale;
  int32_t M, pos0, heads, dim_p, rot_p, lat_p, vdim, vdim_p, key_blocks, ldo, dtype;
} ti_latent_prefill_args;
int ti_latent_attn_prefill(const ti_latent_prefill_args* a, ti_stream_t s);

/* ------------------------------------------------------------------- grouped-query attention
 * A stream slot's cache holds, per key/value head, blocks of 64 positions, each a run of MFMA fragments:
 *   [key tile 4][dim_p / KT][64][VEC] keys, then [vdim_p / 16][64 / KT][64][VEC] values, transposed
 * (value fragment element t * 4 + r of lane group g is position t * 16 + 4 g + r of its KT span).
 * dim_p = dim rounded up to KT, vdim_p to 16; ti_gqa_block_elems elements a block.
 *
 * ti_gqa_prep: per row, from the fused projection a32 [M][lda] fp32 (queries at 0, keys at k_off, values
 * at v_off; k_off < 0: no keys and values, the layer reads another's cache):
 *   q T [M][heads][dim_p] = rms_norm(all query rows; q_w) * (q_scale ? q_scale[pos] : 1)
 *   cache position pos[m] = rms_norm(all key rows; k_w), values. */
typedef struct ti_gqa_prep_args {
  const float* a32;
  int32_t lda, M, heads, kv_heads, dim, vdim, k_off, v_off;
  const float* q_w;
  const float* k_w;
  const float* q_scale;        /* nullable [position]                                        */
  const int32_t* pos;
  const int32_t* slot;         /* nullable [M]: stream slot of row m (NULL: m)               */
  void* q;
  void* cache;
  int64_t slot_stride;         /* elements; 0: all rows share one slot (prompt chunk)        */
  int32_t seq_p;               /* positions a slot holds, a multiple of 64                   */
  float eps;
  int32_t dtype;
} ti_gqa_prep_args;
int ti_gqa_prep(const ti_gqa_prep_args* a, ti_stream_t s);
int ti_gqa_block_elems(int dtype, int dim, int vdim);

/* Attention of rows [0, M) over cache positions [0, pos[m]] of their slots: scores * scale, softmax whose
 * denominator also holds exp(sink[h]) (sink NULL: not), values, times sigmoid(gate[m][h * vdim + d])
 * (gate NULL: 1); out T [M][ldo].  Query head h reads key/value head h / (heads / kv_heads).
 * ti_gqa_decode: any rows; keys split over `splits` (ti_gqa_splits) workgroups, more than one: part_o fp32
 * [M][splits][heads][vdim_p] and part_ml fp32 [M][splits][heads][2] are merged by a second launch.
 * ti_gqa_prefill: consecutive positions pos0 + m of one slot (slot_stride 0). */
typedef struct ti_gqa_attn_args {
  const void* q;
  const void* cache;
  int64_t slot_stride;
  const int32_t* pos;
  const int32_t* slot;
  const float* sink;
  const float* gate;
  void* out;
  float* part_o;
  float* part_ml;
  float scale;
  int32_t M, pos0, heads, kv_heads, dim, vdim, seq_p, splits, ldg, ldo, dtype;
} ti_gqa_attn_args;
int ti_gqa_decode(const ti_gqa_attn_args* a, ti_stream_t s);
int ti_gqa_prefill(const ti_gqa_attn_args* a, ti_stream_t s);
int ti_gqa_splits(int M, int heads, int kv_heads, int max_seq);
/* Once per process and device, before a capture: lifts the LDS limit of the kernels of this and the
 * next section. */
int ti_recurrent_prepare(void);

/* ------------------------------------------------------------------- short convolution
 * Causal convolution per channel over a prompt chunk (rows: consecutive positions of slot `slot0`):
 * y[c] = b[c] + sum_j w[j][c] x[position - (taps - 1) + j][c], zeros before position 0, through `act`
 * (TI_CONV_*).  A slot's last inputs live in a ring [taps][channels] T, position p at place p % taps; the
 * chunk's first rows read it, and it is left as it is (ti_ssd_norm / ti_lru_scan write it).
 * Output place of channel c: c for c < c0, else o0 + (c - c0) / bw * bwp + (c - c0) % bw; the places a
 * section of bw channels leaves free are zeroed. */
enum ti_conv_act { TI_CONV_LINEAR = 0, TI_CONV_SILU = 1 };
typedef struct ti_conv_args {
  const void* x;               /* T [M][ldx]                                                 */
  const void* ring;            /* T [slots][taps][channels]                                  */
  const float* w;              /* [taps][channels]                                           */
  const float* b;
  void* out;                   /* T [M][ldo]                                                 */
  const int32_t* pos;
  int32_t M, channels, taps, act, ldx, ldo, c0, o0, bw, bwp, slot0, dtype;
} ti_conv_args;
int ti_conv(const ti_conv_args* a, ti_stream_t s);

/* ------------------------------------------------------------------- state-space recurrence (SSD)
 * dt = softplus(dt_raw + dt_bias); S = exp(-exp(a_log) dt) S + dt B x^T; y = S^T C + D x, per head, fp32.
 * A slot's state is [heads][vdim][np] fp32, np = state rounded up to 4; zero before position 0.
 * ti_ssd_step: one token per row, each row its own slot; x, B, C come from the raw projection
 * [z inner | x inner | B groups * state | C groups * state] T through the short convolution (SiLU), whose
 * ring it advances.
 * ti_ssd_scan: a prompt chunk of slot `slot0`; x, B, C come convolved from ti_conv's output: x at 0, B of
 * group g at o0 + g * nk, C behind all B, nk = state rounded up to KT. */
typedef struct ti_ssd_args {
  const void* a;               /* step: T [M][lda] raw projection; scan: T [M][lda] convolved */
  const float* dt;             /* [M][heads] raw                                             */
  const float* dt_bias;
  const float* a_log;
  const float* d;
  const float* conv_w;         /* step: [taps][channels]                                     */
  const float* conv_b;
  void* ring;
  float* state;
  float* y;                    /* [M][ldy]                                                   */
  const int32_t* pos;
  const int32_t* slot;
  int32_t M, heads, vdim, state_n, groups, taps, lda, ldy, o0, slot0, dtype;
} ti_ssd_args;
int ti_ssd_step(const ti_ssd_args* a, ti_stream_t s);
int ti_ssd_scan(const ti_ssd_args* a, ti_stream_t s);

/* Gate before the norm: v = y * silu(z), RMS norm in `groups` equal parts, times w; out T [M][ldo].
 * ring non-NULL (prompt chunk): the last taps - 1 rows' convolution inputs (raw + inner) enter it. */
typedef struct ti_ssd_norm_args {
  const float* y;              /* [M][ldy]                                                   */
  const void* raw;             /* T [M][lda], z at 0                                         */
  const float* w;
  void* out;
  void* ring;
  const int32_t* pos;
  float eps;
  int32_t M, inner, groups, lda, ldy, ldo, channels, taps, slot0, dtype;
} ti_ssd_norm_args;
int ti_ssd_norm(const ti_ssd_norm_args* a, ti_stream_t s);

/* ------------------------------------------------------------------- linear recurrence over a chunk
 * S = a S + b per channel over the rows of a prompt chunk (TI_DE_LRU pairs), out T [m][c] = S * y[m][c];
 * the slot's state [channels] fp32 (zero before position 0) and convolution ring (inputs x) are advanced. */
typedef struct ti_lru_scan_args {
  const float* ab;             /* [M][channels][2]                                           */
  const void* y;               /* T [M][ldy]                                                 */
  const void* x;               /* T [M][ldy]                                                 */
  void* out;                   /* T [M][ldo]                                                 */
  float* state;                /* [slots][channels]                                          */
  void* ring;
  const int32_t* pos;
  int32_t M, channels, taps, ldy, ldo, slot0, dtype;
} ti_lru_scan_args;
int ti_lru_scan(const ti_lru_scan_args* a, ti_stream_t s);

/* One token per row of a gated linear recurrent unit, each row its own slot: the row's convolution (inputs
 * x and the ring, which it advances), the block-diagonal gate products and the step S = a S + b of TI_DE_LRU,
 * out T [m][c] = S * y[m][c].  gates: fragment-ordered [blocks][2 * width / blocks] rows (recurrence, input)
 * per channel; gate_b in the same order. */
typedef struct ti_lru_step_args {
  const void* x;               /* T [M][ldx]                                                 */
  const void* y;               /* T [M][ldx]                                                 */
  void* ring;
  const float* conv_w;         /* [taps][channels]                                           */
  const float* conv_b;
  const void* gates;
  const float* gate_b;
  const float* lru_rate;       /* [channels]                                                 */
  float* state;                /* [slots][channels]                                          */
  void* out;                   /* T [M][ldo]                                                 */
  const int32_t* pos;
  const int32_t* slot;         /* nullable [M]: stream slot of row m (NULL: m)               */
  int32_t M, channels, blocks, taps, ldx, ldo, dtype;
} ti_lru_step_args;
int ti_lru_step(const ti_lru_step_args* a, ti_stream_t s);
int ti_lru_step_max_block(int dtype);   /* most channels a block may have */

/* Seeded uniform(-scale, scale) elements of `dtype` (synthetic weights and caches). */
int ti_stack_fill(uint64_t seed, uint32_t tid, uint64_t n, float scale, int dtype, void* out, ti_stream_t s);

#ifdef __cplusplus
}
#endif
#endif /* TI_STACK_H */
