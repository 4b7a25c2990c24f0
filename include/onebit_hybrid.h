/*
 * onebit_hybrid.h -- C ABI of the hybrid decoders of libonebit_hybrid.so: dense-weight decoder-only models whose layers mix sigmoid
 * attention and state-space recurrences, each next to a gated feed-forward that reads the same norm.
 *
 * A layer is two matrix products around its mixer:
 *   h   = rms_norm(x)                                              fp32 residual x
 *   [mixer inputs | auxiliary fp32 columns | gate, up] = W_in h    (mixer projections and feed-forward share the input: one product)
 *   x  += mult * ([mixer output | silu(gate) * up] W_out^T + b)    (... and the output: one product over the concatenated columns)
 * Both weight matrices are packed once, FRAGMENT-MAJOR (onebit_amd/csrc/ob_dense.h): tiles of 16 rows x 64 bytes, 1 KB each.
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

#define ONEBIT_HYBRID_ABI_VERSION 1
#define ONEBIT_HYB_BF16 2          /* operands bf16, accumulation and everything listed as fp32 in fp32 */
#define ONEBIT_HYB_F32  1          /* everything fp32 */

#define ONEBIT_MIX_SIGMOID_ATTENTION 0
#define ONEBIT_MIX_SSM               1

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
} onebit_hlayer_t;

typedef struct onebit_hrun {     /* one pass over a layer; a repeated layer appears once per repetition                        */
    int32_t layer, add_embedding;
    void *s0, *s1;               /* attention: k [slots][kv_heads][max_len][kp], v [..][vp]; state space: fp32 state
                                    [slots][heads][state][sp], convolution ring [slots][taps][channels]                          */
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
} onebit_hmodel_t;

typedef struct onebit_hseg { int32_t row0, n, slot, past; } onebit_hseg_t;

typedef struct onebit_hstate {
    uint64_t struct_size;
    int32_t n_rows, n_dec, n_seg, n_out;         /* rows 0 .. n_dec - 1: one token each; prompt chunks tile the rest             */
    int32_t attn_chunk, attn_splits;             /* decode attention: positions per workgroup (multiple of 128), workgroups per
                                                    head; chunk * splits >= the longest context of the decode rows               */
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
