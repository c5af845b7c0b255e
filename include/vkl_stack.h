/*
 * C ABI of decoder stacks whose layers differ from one another (in
 * libvkllama_hip.so): bf16 weights, an fp32 residual stream, layers with one
 * norm whose output feeds the token mixer and the feed-forward part in
 * parallel, or with a norm for each, one after the other; mixers whose values
 * are their keys (attention over shared key/value rows, latent attention, where
 * the shared row is the normed latent of a token), attention with rotated and
 * normed keys within chunks, and linear recurrences (the gated delta rule, sums
 * that decay).  No counterpart in the reference, which runs Llama-2 blocks only.
 *
 * Two number formats (`type` arguments, GGML numbers):
 *   30 BF16: matrix products and stored activations in bf16 with fp32 sums
 *    0 F32:  activations, caches and products in true 32-bit
 * Weights are bf16 in both.  In both, positions, attention scores and weights,
 * norms, gates and the residual stream are fp32.
 *
 * Conventions are those of vkl_hip.h.  Row sizes: a row that a product reads
 * is padded with zeros to a multiple of 64 values, a head to a multiple of 32.
 */
#ifndef VKL_STACK_H
#define VKL_STACK_H
#include <stddef.h>
#include <stdint.h>

#ifdef __cplusplus
extern "C" {
#endif

#define VKL_TYPE_F32 0
#define VKL_TYPE_BF16 30

/* activations of a product's outputs */
#define VKL_ACT_NONE 0
#define VKL_ACT_SILU 1
#define VKL_ACT_RELU2 2 /* the square of relu */
#define VKL_ACT_GELU 3  /* z times the normal distribution function of z (erf) */

/* ---- operators (any number of token rows) -------------------------------- */

/* The output columns of a product fall into segments, each with its own
 * destination: projections that share an input are one matrix. */
typedef struct
{
  int n0;                /* first column (row of w), a multiple of 8 */
  int n;                 /* columns written; up to the next segment: padding */
  void *y;               /* [M, n], row stride ys (elements) */
  size_t ys;
  int type;              /* VKL_TYPE_F32 or VKL_TYPE_BF16 */
  int act;               /* VKL_ACT_... */
  const float *residual; /* F32 only, layout of y: y = residual + v */
  float cap;             /* > 0: y = cap * tanh (v / cap) */
} vkl_out_seg;

/* y = x W^T, W bf16 [N, K], K % 64 == 0, at most 4 segments.  x bf16: matrix
 * cores; x fp32: products and sums in 32-bit. */
int vkl_project_bf16w (const void *x, int xtype, size_t xs, const void *w,
                       int M, int N, int K, const vkl_out_seg *segs, int nseg,
                       void *stream);
/* out[i, :W] = rms_norm (table[toks[i]]) * w (w null: the plain rows), fp32 rows
 * of stride os; table bf16 [VH, K] of which the first W columns are valid;
 * ids >= VH read row 0.  Columns W .. os-1 are not written. */
int vkl_embed_norm_bf16 (const void *table, uint32_t VH, int K, int W,
                         const uint32_t *toks, uint32_t n, const float *w,
                         float eps, float *out, size_t os, void *stream);
/* out[i, :W] = table[toks[i]] * scale, otherwise as above */
int vkl_embed_rows_bf16 (const void *table, uint32_t VH, int K, int W,
                         const uint32_t *toks, uint32_t n, float scale,
                         float *out, size_t os, void *stream);
/* out[i, :W] = x[r] / sqrt (mean (x[r]^2) + eps) * w for r = rows ? rows[i] : i;
 * columns W .. Wp-1 of out are set to zero */
int vkl_rmsnorm_f32 (const float *x, size_t xs, const uint32_t *rows, int n,
                     int W, const float *w, float eps, void *out, int otype,
                     size_t os, int Wp, void *stream);
/* Causal attention of many query rows on the matrix cores, bf16: q [S, H*hd],
 * k and v [L, G*hd] (they may be the same rows), query head h reads head
 * h / (H/G); query row s is at position s + L - S and its scores are
 * q.k * scale * (1 + temp_coef * ln (floor ((p + 1) / temp_every) + 1)); gate:
 * optional fp32 [S, gs], head h's output times sigmoid (gate[s, h]).  hd a
 * multiple of 32 up to 256. */
int vkl_attn_prefill_causal_bf16 (const void *q, const void *k, const void *v,
                                  int H, int G, int S, int L, int hd,
                                  size_t qhs, size_t khs, size_t vhs,
                                  float scale, float temp_coef, int temp_every,
                                  const float *gate, size_t gs, void *out,
                                  size_t ors, void *stream);
/* The same where the values ARE the keys, for few query rows (decode) and for the
 * 32-bit format: q [S, H*dim] and out in qtype / otype, rows [>= pos0 + S, G*dim]
 * in ctype; query row s is at position pos0 + s.  One pass over the rows.  bf16
 * rows that several heads share go through the matrix cores (queries and
 * weights rounded to bf16 as operands), others through the vector units in fp32
 * throughout.  The context is split over workgroups, the last of which combines
 * the parts (scratch from vkl_attn_rows_scratch_bytes, zeroed once).  dim a
 * multiple of 32 up to 1024. */
int vkl_attn_rows (const void *q, int qtype, size_t qs, const void *rows,
                   int ctype, size_t rs, int H, int G, int dim, int S,
                   uint32_t pos0, float scale, float temp_coef, int temp_every,
                   void *out, int otype, size_t os, void *scratch,
                   void *stream);
size_t vkl_attn_rows_scratch_bytes (int ctype, int H, int G, int dim, int S);
/* What happens to queries, keys and values between their projections and the
 * attention.  Queries and keys: rotation of the pairs (i, i + npair) by
 * position * freq[i], then an RMS norm over `n` values without weights.
 * Values: (1 - mix) v + mix * first (first null: v as it is).  All in fp32.
 * A null source skips its part; source and destination may be the same rows.
 * Heads lie `dim` values apart, of which the first n (values: all) count, the rest
 * of a query or key is set to zero. */
typedef struct
{
  int H, G, dim, n;
  int npair;             /* pairs that are rotated; 0: none */
  const double *freq;    /* [npair], device */
  float eps;
  const void *q;         /* [S, H*dim], row stride qs, in qtype */
  size_t qs;
  void *qo;
  size_t qos;
  int qtype, qotype;
  const void *k, *v;     /* [S, G*dim], row stride kvs, in kvtype */
  size_t kvs;
  int kvtype;
  void *ko, *vo;         /* rows of the caches, stride G*dim, in ctype: the row of position 0 */
  const void *first;     /* such rows of another layer's values, in ctype, its heads
                            fdim apart (as many heads; beyond fdim: zeros) */
  int fdim;
  float mix;
  int ctype;
} vkl_attn_rows_prep;
int vkl_attn_prepare (const vkl_attn_rows_prep *p, int S, uint32_t pos0,
                      void *stream);
/* Attention over keys and values of their own, few query rows or fp32; as
 * vkl_attn_rows, and: rows are keys, vals values (same strides); chunk > 0: a
 * position sees those before it from the last multiple of chunk on; sink: the
 * softmax has one more score, 0, without a value. */
int vkl_attn_kv_rows (const void *q, int qtype, size_t qs, const void *rows,
                      const void *vals, int ctype, size_t rs, int H, int G,
                      int dim, int S, uint32_t pos0, float scale, int chunk,
                      int sink, void *out, int otype, size_t os,
                      void *scratch, void *stream);
size_t vkl_attn_kv_rows_scratch_bytes (int ctype, int H, int G, int dim, int S);
/* the same for many query rows on the matrix cores, bf16; shapes as for
 * vkl_attn_prefill_causal_bf16 */
int vkl_attn_prefill_chunked_bf16 (const void *q, const void *k, const void *v,
                                   int H, int G, int S, int L, int hd,
                                   size_t qhs, size_t khs, size_t vhs,
                                   float scale, int chunk, int sink, void *out,
                                   size_t ors, void *stream);

/* ---- linear recurrences ---------------------------------------------------- */
/* Causal convolution over time per channel, then SiLU: out[s, c] = silu (sum_j
 * w[c, taps-1-j] x(s - j)[c]) with x of the positions before pos0 from ring (the
 * row of position p is p % taps, fp32 [taps, n]; zeros before position 0), which
 * afterwards holds the last inputs.  n a multiple of 8, taps 1 .. 16; x and out in
 * `type`, w fp32 [taps, n], row j meeting the token taps-1-j before. */
int vkl_short_conv_silu (const void *x, int type, size_t xs, const float *w,
                         int n, int taps, float *ring, uint32_t pos0, int S,
                         void *out, size_t os, void *stream);
/* Per head a state M [dim, vdim], zero before position 0:
 *   gated delta rule (b given): with q, k made unit vectors
 *     (x / sqrt (sum x^2 + unit_eps)), q also times qscale,
 *     M <- diag (g) M,  u = beta (v - M^T k),  M <- M + k u^T,  out = M^T q,
 *     g = exp (-rate[h] softplus (z + dt_bias)), beta = sigmoid (b),
 *     z given, or (chunked form only) z = a1 w_a2^T of low rank
 *   decaying sums (b null): M <- exp (log_decay[h]) M + k v^T,  out = M^T q * qscale
 * Everything after q, k, v, z (a1) and b is fp32.  Head h reads query/key head
 * h / rep.  dim and vdim are multiples of 32 up to 256, heads lie as densely. */
typedef struct
{
  int H, rep, dim, vdim;
  const void *q, *k, *v; /* [S, H/rep*dim], the same, [S, H*vdim] in `type` */
  int type;
  size_t qs, ks, vs;     /* row strides, multiples of 8 */
  float qscale;
  const float *log_decay; /* [H] */
  const float *z;         /* [S, H*dim], row stride zs (a multiple of 4) */
  size_t zs;
  const void *a1;         /* [S, r_a] in `type`, row stride as (a multiple of 8) */
  size_t as;
  const void *w_a2;       /* bf16 [H*dim, r_a], r_a a multiple of 64 */
  int r_a;
  const float *b;         /* [S, H], row stride bs */
  size_t bs;
  const float *dt_bias;   /* [H*dim] */
  const float *rate;      /* [H] */
  float unit_eps;
  float *state;           /* [H, dim, vdim] */
  float *out;             /* [S, H*vdim], row stride os */
  size_t os;
} vkl_recurrence_args;
/* form: VKL_RECUR_TOKENS one token after the other; VKL_RECUR_CHUNKS 64 at a time
 * as matrix products (dim up to 128); VKL_RECUR_AUTO by S and dim */
#define VKL_RECUR_AUTO 0
#define VKL_RECUR_TOKENS 1
#define VKL_RECUR_CHUNKS 2
int vkl_recurrence (const vkl_recurrence_args *a, int S, uint32_t pos0,
                    int form, void *scratch, size_t scratch_bytes,
                    void *stream);
/* whether VKL_RECUR_AUTO takes the chunked form (it needs scratch memory then) */
int vkl_recurrence_chunked (const vkl_recurrence_args *a, int S);
/* what the chunked form needs for S tokens at once (it takes them in pieces if
 * there is less, at least what 64 tokens need) */
size_t vkl_recurrence_scratch_bytes (const vkl_recurrence_args *a, int S);
/* out = x / sqrt (mean of a group's x^2 + eps) * w * sigmoid (gate): groups of gw
 * neighbouring values of which n count in the mean (the others are zero);
 * x fp32; w fp32, [gw] shared by the groups; gate and out in `type` */
int vkl_gated_norm (const float *x, size_t xs, int groups, int gw, int n,
                    const float *w, float eps, const void *gate, size_t gs,
                    int type, int S, void *out, size_t os, void *stream);

/* the same per head of vdim values (a multiple of 32 up to 256, n of them valid)
 * with gates of low rank: gate = g1 g2^T, g1 [S, r] in `type`, row stride gs, g2 bf16
 * [H*vdim, r], r a multiple of 64; w [vdim] */
int vkl_low_rank_gated_norm (const float *x, size_t xs, int H, int vdim, int n,
                             const float *w, float eps, const void *g1,
                             size_t gs, const void *g2, int r, int type, int S,
                             void *out, size_t os, void *stream);

/* ---- per-head products ------------------------------------------------------ */
/* y[s, h*yh + r] = f * sum_k w[h, r, k] x[s, h*xh + k], w bf16 [H, R, K], f = 1 or
 * sigmoid (gate[s*gs + h]); K a multiple of 32 */
int vkl_head_matvec (const void *w, int H, int R, int K, const void *x,
                     int xtype, size_t xs, size_t xh, void *y, int ytype,
                     size_t ys, size_t yh, const float *gate, size_t gs, int S,
                     void *stream);

/* ---- the one-token step ---------------------------------------------------- */
/* mixers */
#define VKL_MIX_SHARED_KV 0 /* q.k over rows that are keys and values */
#define VKL_MIX_LATENT 1    /* q -> W_uk^T q, attention over latents, W_uv */
#define VKL_MIX_KV 2        /* rotated, normed q.k over keys, values of their own */
#define VKL_MIX_DELTA 3     /* short convolutions, gated delta rule, gated norm */
#define VKL_MIX_DECAY 4     /* decaying sums, gated norm over all heads */

/* One layer run: a layer that runs several times appears once per run, with
 * the same weights and a cache of its own. */
typedef struct
{
  int mixer;
  int H, G;             /* query heads, key/value heads (latent: 1) */
  int dim, vdim;        /* padded head sizes of queries/keys and values */
  int rank, rank_p;     /* latent size, padded (latent) */
  float scale, temp_coef;
  int temp_every;
  int ff;               /* feed-forward rows, 0: none */
  const float *norm;    /* [width_p] */
  const void *w_in;     /* bf16 [n_in, width_p]: q | k or down-projection | gate | up */
  int n_in;
  int kv0, g0, up0;     /* first rows of those parts (multiples of 8); q at 0 */
  const void *w_out;    /* bf16 [width, k_out]: columns of the heads | feed-forward */
  int k_out, ff_col;
  const void *w_ukt;    /* latent: bf16 [H, rank_p, dim] (transposed) */
  const void *w_uv;     /* latent: bf16 [H, vdim, rank_p] */
  const float *c_norm;  /* latent: [rank_p] */
  void *cache;          /* [maxlen, G*dim] or [maxlen, rank_p] */

  /* a layer with two norms: the feed-forward part has a norm and an input of its
   * own.  norm2 null: the parallel form (or no feed-forward part, ff 0). */
  const float *norm2;   /* [width_p] */
  const void *w_up;     /* bf16 [ff rounded up to 8, width_p] */
  const void *w_down;   /* bf16 [width, ff_p] */
  int ff_p, ff_act;     /* ff_p a multiple of 64 */

  /* VKL_MIX_KV: w_in rows q | k (kv0) | v (v0) */
  int v0, n, npair, chunk, sink; /* as in the operators above; n: head size without padding */
  const double *freq;
  void *vcache;         /* [maxlen, G*dim] */
  const void *vfirst;   /* values cache of another layer, or null */
  int fdim;             /* head size of its rows */
  float vmix;

  /* VKL_MIX_DELTA: w_in rows q | k (kv0) | v (v0), convolved, | b (b0) | a1 (a0) |
   * g1 (g0).  VKL_MIX_DECAY: q | k | v | gate (g0).  G: query/key heads */
  int b0, a0, taps, vn; /* vn: value head size without padding */
  int r_a, r_g;         /* columns of w_a2 and w_g2, multiples of 8 */
  const void *w_a2, *w_g2; /* bf16 [H*dim, r_a], [H*vdim, r_g] */
  const float *conv;    /* [taps, (2 G dim + H vdim)] */
  float *ring;          /* the same shape */
  const float *dt_bias, *rate, *log_decay, *gnorm; /* gnorm: [vdim] or [H*vdim] */
  float qscale, unit_eps;
  float *state;
} vkl_stack_layer;

typedef struct
{
  int width, width_p, vocab, maxlen, n_runs;
  int ctype;             /* type of the caches */
  float eps, logit_cap;  /* logit_cap 0: none */
  const vkl_stack_layer *layers_h; /* HOST array [n_runs] */
  const void *embed;     /* bf16 [vocab, width_p] */
  const void *head;      /* output matrix, as embed; null: embed */
  float embed_scale;     /* without embed_norm */
  const float *embed_norm, *final_norm; /* [width_p]; embed_norm may be null */
  void *scratch;         /* vkl_stack_scratch_bytes, zeroed once */
} vkl_stack_model;

size_t vkl_stack_scratch_bytes (const vkl_stack_model *m);
/* 1 if the step covers this model (rows of up to 32768 values, sizes padded as
 * above), else 0; the operators above serve every model */
int vkl_stack_supported (const vkl_stack_model *m);
/* One token at position pos: 3 launches per parallel shared-row layer (norm + all
 * projections; attention; output + feed-forward + residual), 5 per latent one; a
 * layer with two norms takes 2 (norm + up + activation; down + residual) for the
 * feed-forward part and 3 (recurrences) or 4 (keys and values) for the mixer.
 * Arguments as for vkl_decode_step. */
int vkl_stack_step (const vkl_stack_model *m, const uint32_t *tok,
                    uint32_t pos, float *logits32, uint32_t *next_tok,
                    void *stream);
/* vkl_decode_loop / vkl_decode_loop_sampled for such a stack */
int vkl_stack_loop (const vkl_stack_model *m, uint32_t *ids, uint32_t pos0,
                    int n_steps, float *logits32, void *stream);
int vkl_stack_loop_sampled (const vkl_stack_model *m, uint32_t *ids,
                            uint32_t pos0, int n_steps, float *logits32,
                            int topk, float topp, uint64_t seed, void *stream);
/* drops the captured step of this model, if there is one */
void vkl_stack_release (const vkl_stack_model *m);

#ifdef __cplusplus
}
#endif
#endif
