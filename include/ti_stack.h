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
  TI_DE_VFRAG        /* rows are keys, columns (head, head_w): transposed value fragments,
                        out T [head][head_w / 16][key / KT][64][VEC] (ti_latent_attn_prefill) */
};

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
} ti_dense_args;
int ti_dense(const ti_dense_args* a, ti_stream_t s);
size_t ti_dense_args_bytes(void);

/* ------------------------------------------------------------------- norms and residual
 * One row per workgroup:
 *   y' = post_w ? norm(y; post_w, post_b) : y           (y: fp32 rows, or the weighted expert outputs
 *   x  = x + y'                                          sum_k part_w[m][k] * parts[m * top + k])
 *   xn = T(norm(x; w, b))  and / or  cat = T([x ; x0])
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
  const float* w;              /* nullable: no xn                                            */
  const float* b;
  void* xn;                    /* T [M][ldn]                                                 */
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

/* Seeded uniform(-scale, scale) elements of `dtype` (synthetic weights and caches). */
int ti_stack_fill(uint64_t seed, uint32_t tid, uint64_t n, float scale, int dtype, void* out, ti_stream_t s);

#ifdef __cplusplus
}
#endif
#endif /* TI_STACK_H */
