/*
 * onebit_hybrid.h -- C ABI of the hybrid decoders of libonebit_hybrid.so: dense-weight decoder-only models whose layers mix sigmoid
 * attention, latent attention and state-space recurrences with dense, gated or mixture-of-experts feed-forwards.
 *
 * A PARALLEL layer is two matrix products around its mixer:
 *   h   = rms_norm(x)                                              fp32 residual x
 *   [mixer inputs | auxiliary fp32 columns | gate, up] = W_in h    (mixer projections and feed-forward share the input: one product)
 *   x  += mult * ([mixer output | silu(gate) * up] W_out^T + b)    (... and the output: one product over the concatenated columns)
 * A SEQUENTIAL layer is mixer and feed-forward one after the other, each with optional norms on its input and on its output:
 *   x += mult * post1(mixer(pre1(x)));  x += mult * post2(ff(pre2(x)));  then, if it has one, the token's own input:
 *   x += rms(proj(gelu_tanh(gate x) * e[token])) * w;  and, if it has one, a depth average  x = sum_j dwa[j] X_j  over the embedding
 *   output X_0 and the results X_1 .. of all layers so far.  norm(v, w) = v / sqrt(mean v^2 + eps) * w.
 * All weight matrices are packed once, FRAGMENT-MAJOR (onebit_amd/csrc/ob_dense.h): tiles of 16 rows x 64 bytes, 1 KB each.
 *
 * Conventions of onebit.h: device pointers owned by the caller, stream-ordered, no allocation, no synchronisation, graph-capture
 * safe; 0 = ok, negative = argument error (ONEBIT_E_*), positive = hipError_t; onebit_hybrid_last_error() has the message.
 */
#ifndef ONEBIT_HYBRID_H
#define ONEBIT_HYBRID_H
#include <stddef.h>
#include <stdint.h>
#ifdef __cplusplus
extern "C" {
#endif

#define ONEBIT_HYBRID_ABI_VERSION 2
#define ONEBIT_HYB_BF16 2          /* operands bf16, accumulation and everything listed as fp32 in fp32 */
#define ONEBIT_HYB_F32  1          /* everything fp32 */
#define ONEBIT_HYB_SHORT 16        /* rows of a short prompt chunk */

#define ONEBIT_MIX_SIGMOID_ATTENTION 0
#define ONEBIT_MIX_SSM               1
#define ONEBIT_MIX_LATENT_ATTENTION  2

#define ONEBIT_LAYER_PARALLEL        0
#define ONEBIT_LAYER_SEQUENTIAL      1

/* latent attention (csrc/ob_latent.h).  w_in = [W_dq | W_dkv], the second from n tile nt_q on; no bias */
typedef struct onebit_hlatent {
    int32_t q_rank, kv_rank, nt_q;
    int32_t rp;                  /* kv_rank padded: columns of a cached row (bf16 tiled form: 64, 128, 256 or 512)                */
    int32_t tiled;               /* bf16 MFMA decode form                                                                          */
    int32_t flash;               /* prompts expanded to keys and values of kp = vp = 64 or 128 columns, or 0                       */
    int32_t vdp;                 /* value columns per head in w_out and w_uv (vdim rounded up to 32)                               */
    const float *qn_w, *kvn_w;   /* [q_rank], [kv_rank]                                                                            */
    const void *w_uq;            /* [heads kp rows][q_rank]: head by head, kp rows each                                           */
    const void *w_uk;            /* [heads rp rows][kp]: per head the transposed key projection                                   */
    const void *w_uv;            /* [heads vdp rows][rp]                                                                           */
    const void *w_kv;            /* flash: [2 heads kp rows][rp]: keys of all heads, values of all heads                           */
} onebit_hlatent_t;

/* feed-forward of a sequential layer: any of a plain part (xIELU), a gated part (also a shared expert) and routed experts */
typedef struct onebit_hff {
    int32_t nt_plain;            /* n tiles of w_plain_in (even), 0: none.  ff(h) = W_out xielu(W_in h)                            */
    int32_t nt_gated;            /* n tiles of gate / up in w_gated_in behind the nt_aux router tiles (multiple of 4), 0: none     */
    int32_t nt_aux;              /* router: n tiles of experts + identity fp32 logits (even)                                       */
    int32_t nt_expert;           /* n tiles of gate / up of one expert (multiple of 4)                                             */
    int32_t experts, identity, top, groups, keep;
    float act_a, act_b;          /* xIELU: a z^2 + z / 2 above zero, b (e^z - 1 - z) + z / 2 below                                */
    const void *w_plain_in, *w_plain_out, *w_gated_in, *w_gated_out, *w_expert_in, *w_expert_out;   /* experts one after the other */
    const float *correction;     /* [experts + identity]                                                                           */
} onebit_hff_t;

typedef struct onebit_hside {    /* the token's own input to a sequential layer */
    int32_t dim, nt;             /* nt: n tiles of w_gate (even), 0: none                                                          */
    const void *w_gate, *w_proj;
    const float *norm_w;
    const void *table;           /* first column of this layer's part of the token table (row-major, side_cols columns)            */
} onebit_hside_t;

typedef struct onebit_hlayer {
    int32_t kind;                /* ONEBIT_MIX_*                                                                                */
    int32_t nt_mix, nt_aux;      /* 16-column tiles of the mixer's columns / of its fp32 columns (their sum even)                */
    int32_t nt_in;               /* all n tiles of w_in: nt_mix + nt_aux + 2 ceil(ff / 16)                                       */
    int32_t mix_k, act_k;        /* padded columns of w_out's two parts (multiples of the tile width); act_k = 0: no feed-forward */
    const void *w_in, *w_out;    /* fragment-major [nt_in][width_pad / KT] and [ceil(width / 16)][(mix_k + act_k) / KT]          */
    const float *b_in, *b_out;   /* fp32 [16 nt_mix] / [width], or NULL                                                          */
    const float *norm_w;         /* fp32 [width]                                                                                 */
    int32_t heads, vdim;
    /* attention: columns [q: heads dim | k: kv_heads dim | v: kv_heads vdim] */
    int32_t kv_heads, dim, kp, vp, unit_rms;      /* kp, vp: padded head sizes of the cache                                      */
    float scale;
    const float *r1, *r2, *pb;   /* fp32 [heads] or NULL                                                                         */
    /* state space: columns [z: heads vdim | x: heads vdim | B: groups state | C: groups state], auxiliary column h = raw dt       */
    int32_t groups, state, taps, norm_groups, sp; /* sp: vdim rounded up to 4                                                     */
    const float *conv_w, *conv_b, *dt_bias, *A_log, *D, *gnorm_w;     /* conv_w [taps][channels]                                  */
    int32_t form;                /* ONEBIT_LAYER_*; sequential: norm_w is pre1 and may be NULL, act_k = 0, nt_in without feed-forward */
    const float *post1_w, *pre2_w, *post2_w;      /* fp32 [width] or NULL (norms of sequential layers; pre norms use norm_off)    */
    const float *dwa;            /* fp32 [layer runs so far + 1] or NULL                                                           */
    onebit_hlatent_t latent;
    onebit_hff_t ff;
    onebit_hside_t side;
} onebit_hlayer_t;

typedef struct onebit_hrun {     /* one pass over a layer; a repeated layer appears once per repetition                        */
    int32_t layer, add_embedding;
    void *s0, *s1;               /* attention: k [slots][kv_heads][max_len][kp], v [..][vp]; state space: fp32 state
                                    [slots][heads][state][sp], convolution ring [slots][taps][channels]; latent attention: s0 =
                                    rows c, fragment-major [slots][ceil(max_len / 16)][rp / KT] tiles                             */
} onebit_hrun_t;

typedef struct onebit_hmodel {
    uint64_t struct_size;        /* sizeof(onebit_hmodel_t) (checked)                                                            */
    int32_t dtype, width, width_pad, vocab, n_layers, n_runs, n_slots, max_len, max_pos;
    float eps, norm_off, mult, softcap;          /* norm weight = norm_off + w; softcap 0 = none                                  */
    const void *embed, *pos_embed;               /* row-major, dtype; pos_embed [max_pos][width] or NULL                          */
    const float *final_norm;
    const void *head;                            /* fragment-major [ceil(vocab / 16)][width_pad / KT]                             */
    const onebit_hlayer_t *layers;               /* HOST */
    const onebit_hrun_t *runs;                   /* HOST */
    float embed_scale;
    const void *bigram; int32_t buckets, mul_prev, mul_cur;   /* row (previous token mul_prev + token mul_cur) % buckets is added to the embedding;
                                                    row `buckets` at position 0; NULL: none                                       */
    int32_t *token_history;                      /* [n_slots][max_len]: tokens of the slots (state; needed with bigram)           */
    int32_t side_cols;                           /* columns of the token table of the layers' own inputs                          */
} onebit_hmodel_t;

typedef struct onebit_hseg { int32_t row0, n, slot, past; } onebit_hseg_t;

typedef struct onebit_hstate {
    uint64_t struct_size;
    int32_t n_rows, n_dec, n_seg, n_out;         /* rows 0 .. n_dec - 1: one token each; prompt chunks tile the rest             */
    int32_t n_short;                             /* the first n_short chunks may be served like single tokens (each at most
                                                    ONEBIT_HYB_SHORT rows)                                                        */
    int32_t attn_chunk, attn_splits;             /* decode attention: positions per workgroup (multiple of 128), workgroups per
                                                    head; chunk * splits >= the longest context of the decode rows and short chunks */
    const int32_t *tokens, *row_slot, *row_pos, *row_off;    /* device [n_rows]; row_off: tokens of the item before this row;
                                                                row_slot -1 or row_pos -1 = idle row                             */
    const onebit_hseg_t *segs;                   /* HOST [n_seg] */
    const int32_t *out_rows;                     /* device [n_out] */
    float *logits;                               /* fp32 [n_out][vocab] */
    int32_t *next_tokens;                        /* [n_out] greedy tokens, or NULL */
    float *residuals;                            /* optional fp32 [n_runs][n_rows][width]: the residual stream after every run    */
    void *workspace; size_t workspace_bytes;     /* onebit_hybrid_workspace_bytes, 256-byte aligned, ZERO-FILLED ONCE              */
} onebit_hstate_t;

int onebit_hybrid_abi_version(void);
const char *onebit_hybrid_last_error(void);
/* room for steps of up to max_rows rows, max_out sampled rows and max_dec decode rows of max_splits attention splits */
size_t onebit_hybrid_workspace_bytes(const onebit_hmodel_t *m, int64_t max_rows, int64_t max_out, int32_t max_dec, int32_t max_splits);
int onebit_hybrid_step(const onebit_hmodel_t *m, const onebit_hstate_t *s, int64_t max_rows, int64_t max_out, int32_t max_dec,
                       int32_t max_splits, void *stream);
/* z[split][t][n] = W A^T over split's k tiles: the dense product alone (tests, measurements).  n_split splits of ceil(nkt / n_split). */
int onebit_hybrid_gemm(const void *w, const void *a, float *z, int32_t dtype, int32_t n_tiles, int32_t nkt, int32_t T, int32_t n_split, void *stream);
int onebit_hybrid_gemm_splits(int32_t n_tiles, int32_t nkt, int32_t T);

#ifdef __cplusplus
}
#endif
#endif
