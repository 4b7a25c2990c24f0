// Row kernels of the hybrid decoders: the residual stream in fp32 between the two matrix products of a layer, the gated group norm
// behind a recurrent mixer, and the greedy token.
#pragma once
#include "ob_dense.h"

// s += sum of n partial sums `stride` apart: four in flight, added in order
template <int VEC>
__device__ __forceinline__ void ob_sum_splits(float (&s)[VEC], const float *p, size_t stride, int n)
{
    for (int k = 0; k < n; k += 4) {
        float zv[4][VEC];
#pragma unroll
        for (int j = 0; j < 4; ++j)
#pragma unroll
            for (int e = 0; e < VEC; ++e) zv[j][e] = p[(size_t)min(k + j, n - 1) * stride + e];
#pragma unroll
        for (int j = 0; j < 4; ++j)
            if (k + j < n) {
#pragma unroll
                for (int e = 0; e < VEC; ++e) s[e] += zv[j][e];
            }
    }
}

// r = residual row, formed one of two ways; x (fragment-major, the next product's operand) = r / sqrt(mean r^2 + eps) * (off + w)
//   embed != NULL   r = embed[token] (+ pos_embed[position]); copied to emb_save when given
//   else            r = x_in + mult * (sum of the splits of the output product + bias) (+ emb_add: a looped stretch starting over)
// `rows` gathers (the final norm runs on the sampling rows only; the residual is then not written back).
struct ObHNormArgs {
    const void *embed, *pos_embed; const int32_t *tokens, *row_pos;
    float *x; const float *z; size_t z_split; int n_split, ldz; const float *bias; float mult;
    const float *emb_add; float *emb_save;
    const float *w; float off, eps;
    void *out; int out_nkt;
    const int32_t *rows;
    int W;
};

// (the workgroup is as wide as the row allows, up to 1024 threads: at one to 64 rows its few dependent passes ARE the launch's time)
template <typename E, int VEC>
__global__ __launch_bounds__(1024) void ob_hnorm_kernel(const ObHNormArgs A)
{
    extern __shared__ __attribute__((aligned(16))) float sm[];        // [W] row | [16] reduction
    float *red = sm + ((A.W + 3) & ~3);
    const int t = blockIdx.x, tid = threadIdx.x, stride = blockDim.x * VEC;
    const int src = A.rows ? A.rows[t] : t;
    float *xr = A.x + (size_t)src * A.W;
    const E *er = nullptr, *pr = nullptr;
    if (A.embed) {
        er = (const E *)A.embed + (size_t)A.tokens[src] * A.W;
        if (A.pos_embed) pr = (const E *)A.pos_embed + (size_t)max(A.row_pos[src], 0) * A.W;
    }
    float ss = 0.f;
    for (int c = tid * VEC; c < A.W; c += stride) {
        float r[VEC];
        if (er) {
#pragma unroll
            for (int e = 0; e < VEC; ++e) r[e] = (float)er[c + e] + (pr ? (float)pr[c + e] : 0.f);
        } else {
            float s[VEC], xv[VEC];
#pragma unroll
            for (int e = 0; e < VEC; ++e) { s[e] = 0.f; xv[e] = xr[c + e]; }
            ob_sum_splits<VEC>(s, A.z + (size_t)src * A.ldz + c, A.z_split, A.n_split);
#pragma unroll
            for (int e = 0; e < VEC; ++e) r[e] = xv[e] + A.mult * (A.bias ? s[e] + A.bias[c + e] : s[e]);
            if (A.emb_add) {
                const float *ea = A.emb_add + (size_t)src * A.W + c;
#pragma unroll
                for (int e = 0; e < VEC; ++e) r[e] += ea[e];
            }
        }
        if (!A.rows) {
#pragma unroll
            for (int e = 0; e < VEC; ++e) xr[c + e] = r[e];
        }
        if (A.emb_save) {
#pragma unroll
            for (int e = 0; e < VEC; ++e) A.emb_save[(size_t)src * A.W + c + e] = r[e];
        }
#pragma unroll
        for (int e = 0; e < VEC; ++e) { sm[c + e] = r[e]; ss = __builtin_fmaf(r[e], r[e], ss); }
    }
    ss = ob_block_sum(ss, red);
    const float rs = 1.0f / sqrtf(ss / (float)A.W + A.eps);
    E *out = (E *)A.out;
    for (int c = tid * VEC; c < A.W; c += stride) {
        ob_float4 v;
#pragma unroll
        for (int e = 0; e < VEC; ++e) v[e] = sm[c + e] * rs * (A.off + A.w[c + e]);
        if constexpr (VEC == 4) *reinterpret_cast<typename ObElem<E>::V4 *>(out + ob_frag<E>(t, c, A.out_nkt)) = ob_to_v4<E>(v);
        else out[ob_frag<E>(t, c, A.out_nkt)] = (E)v[0];
    }
}

// The same row with everything a sequential layer adds to it:
//   s = sum of the splits (+ bias) + sum_k tok_w[k] ez[tok_row[k]] (experts; eo: their outputs in the work type) + id_w h (identity experts; h = idh or the residual itself)
//   r = x + mult * (post_w ? s / sqrt(mean s^2 + eps) * post_w : s) (+ emb_add)
//     or, embed != NULL: r = embed[token] * embed_scale (+ bigram[row of (previous token, token)]) (+ pos_embed[position])
//   hist: X_i = r is kept (i = hist_i), and with dwa the stream goes on as sum_j dwa[j] X_j, j = 0 .. hist_i
//   output: r / sqrt(mean r^2 + eps) * (off + w), or r itself (w == NULL); fragment-major and, out_rm, also row-major
// The previous token of an item's first row comes from tok_hist [slots][max_len], where every row leaves its token.
struct ObXRowArgs : ObHNormArgs {
    float embed_scale; const void *bigram; int buckets, mul_prev, mul_cur;
    int32_t *tok_hist; const int32_t *row_slot, *row_off; int n_slots, max_len;
    const float *post_w;
    const float *ez; const void *eo; size_t ez_split; int ez_n, ld_ez, top; const int32_t *tok_row; const float *tok_w, *id_w; const void *idh; int ld_idh;
    float *hist; size_t hist_stride; int hist_i; const float *dwa;
    void *out_rm; int ld_rm;
};
// ONE: a thread has one piece of the row (W <= threads * VEC); everything that does not depend on the first reduction is then requested before it.
// KIND: what can be there besides the sum of splits (smaller code: at a few rows a launch's time is its chain of fetches, instructions included)
enum ObXKind { OB_X_PLAIN = 0, OB_X_EXPERTS = 1, OB_X_DEPTH = 2, OB_X_BOTH = 3, OB_X_EMBED = 4 };
template <typename E, int VEC, bool ONE, int KIND>
__global__ __launch_bounds__(1024) void ob_xrow_kernel(const ObXRowArgs A)
{
    constexpr int NH = 8;
    constexpr bool EMB = KIND == OB_X_EMBED, EXP = (KIND & 1) != 0, DEP = (KIND & 2) != 0;
    extern __shared__ __attribute__((aligned(16))) float sm[];        // [W] row | [16] reduction
    float *red = sm + ((A.W + 3) & ~3);
    const int t = blockIdx.x, tid = threadIdx.x, stride = blockDim.x * VEC;
    const int src = A.rows ? A.rows[t] : t;
    float *xr = A.x + (size_t)src * A.W;
    float *hr = A.hist + (size_t)src * A.W;                           // (DEP, and EMB where the embedding is kept)
    const E *er = nullptr, *pr = nullptr, *br = nullptr;
    if constexpr (EMB) {
        const int tok = A.tokens[src], pos = A.row_pos[src], slot = A.row_slot[src];
        er = (const E *)A.embed + (size_t)tok * A.W;
        if (A.pos_embed) pr = (const E *)A.pos_embed + (size_t)max(pos, 0) * A.W;
        if (A.bigram) {
            const bool live = slot >= 0 && slot < A.n_slots && pos >= 0 && pos < A.max_len;
            int b = A.buckets;                                        // (a sequence's first token)
            if (live && pos > 0) {
                const int prev = A.row_off[src] > 0 ? A.tokens[src - 1] : A.tok_hist[(size_t)slot * A.max_len + pos - 1];
                b = (int)(((long long)prev * A.mul_prev + (long long)tok * A.mul_cur) % A.buckets);
            }
            br = (const E *)A.bigram + (size_t)b * A.W;
            if (live && tid == 0 && !A.rows) A.tok_hist[(size_t)slot * A.max_len + pos] = tok;
        }
    }
    float x1[VEC], h1[DEP ? NH : 1][VEC];                             // ONE: the residual and the first results X_j
    if (ONE && !EMB && tid * VEC < A.W) {
#pragma unroll
        for (int e = 0; e < VEC; ++e) x1[e] = xr[tid * VEC + e];
        if (DEP && A.dwa) {
#pragma unroll
            for (int j = 0; j < NH; ++j)
#pragma unroll
                for (int e = 0; e < VEC; ++e) h1[DEP ? j : 0][e] = hr[(size_t)min(j, A.hist_i - 1) * A.hist_stride + tid * VEC + e];
        }
    }
    float ss = 0.f;
    if (!EMB) {
        for (int c = tid * VEC; c < A.W; c += stride) {
            float s[VEC];
#pragma unroll
            for (int e = 0; e < VEC; ++e) s[e] = 0.f;
            if (A.z) ob_sum_splits<VEC>(s, A.z + (size_t)src * A.ldz + c, A.z_split, A.n_split);
            if (A.bias) {
#pragma unroll
                for (int e = 0; e < VEC; ++e) s[e] += A.bias[c + e];
            }
            if (EXP && A.eo) {                                        // four experts in flight, added in order
#pragma unroll 1
                for (int k0 = 0; k0 < A.top; k0 += 4) {
                    float y[4][VEC], w[4];
#pragma unroll
                    for (int j = 0; j < 4; ++j) {
                        const size_t k = (size_t)src * A.top + min(k0 + j, A.top - 1);
                        const int row = A.tok_row[k];                 // (uniform; row 0 where there is none)
                        w[j] = k0 + j < A.top && row >= 0 ? A.tok_w[k] : 0.f;
                        const E *p = (const E *)A.eo + (size_t)max(row, 0) * A.ld_ez + c;
#pragma unroll
                        for (int e = 0; e < VEC; ++e) y[j][e] = (float)p[e];
                    }
#pragma unroll
                    for (int j = 0; j < 4; ++j)
#pragma unroll
                        for (int e = 0; e < VEC; ++e) s[e] = w[j] != 0.f ? __builtin_fmaf(w[j], y[j][e], s[e]) : s[e];
                }
            } else if (EXP) {
#pragma unroll 1
                for (int k0 = 0; k0 < A.top * A.ez_n; k0 += 4) {      // (choice, split) pairs
                    float y[4][VEC], w[4];
#pragma unroll
                    for (int j = 0; j < 4; ++j) {
                        const int kk = min(k0 + j, A.top * A.ez_n - 1), sp = A.ez_n == 1 ? 0 : kk / A.top;
                        const size_t k = (size_t)src * A.top + kk - sp * A.top;
                        const int row = A.tok_row[k];
                        w[j] = k0 + j < A.top * A.ez_n && row >= 0 ? A.tok_w[k] : 0.f;
                        const float *p = A.ez + sp * A.ez_split + (size_t)max(row, 0) * A.ld_ez + c;
#pragma unroll
                        for (int e = 0; e < VEC; ++e) y[j][e] = p[e];
                    }
#pragma unroll
                    for (int j = 0; j < 4; ++j)
#pragma unroll
                        for (int e = 0; e < VEC; ++e) s[e] = w[j] != 0.f ? __builtin_fmaf(w[j], y[j][e], s[e]) : s[e];
                }
            }
            if (EXP && A.id_w) {
                const float w = A.id_w[src];
#pragma unroll
                for (int e = 0; e < VEC; ++e)
                    s[e] = __builtin_fmaf(w, A.idh ? (float)((const E *)A.idh)[(size_t)src * A.ld_idh + c + e] : ONE ? x1[e] : xr[c + e], s[e]);
            }
#pragma unroll
            for (int e = 0; e < VEC; ++e) { sm[c + e] = s[e]; ss = __builtin_fmaf(s[e], s[e], ss); }
        }
    }
    float rp = 1.f;
    if (!EMB && A.post_w) rp = 1.0f / sqrtf(ob_block_sum(ss, red) / (float)A.W + A.eps);          // (uniform)
    ss = 0.f;
    for (int c = tid * VEC; c < A.W; c += stride) {
        float r[VEC];
        if (EMB) {
#pragma unroll
            for (int e = 0; e < VEC; ++e) r[e] = (float)er[c + e] * A.embed_scale + (br ? (float)br[c + e] : 0.f) + (pr ? (float)pr[c + e] : 0.f);
        } else {
#pragma unroll
            for (int e = 0; e < VEC; ++e) r[e] = (ONE ? x1[e] : xr[c + e]) + A.mult * (A.post_w ? sm[c + e] * rp * A.post_w[c + e] : sm[c + e]);
            if (A.emb_add) {
#pragma unroll
                for (int e = 0; e < VEC; ++e) r[e] += A.emb_add[(size_t)src * A.W + c + e];
            }
        }
        if (DEP || (EMB && A.hist)) {
            if (!A.rows) {
#pragma unroll
                for (int e = 0; e < VEC; ++e) hr[A.hist_i * A.hist_stride + c + e] = r[e];
            }
            if (DEP && A.dwa) {
                float a[VEC];
#pragma unroll
                for (int e = 0; e < VEC; ++e) a[e] = 0.f;
                for (int j = 0; j < A.hist_i; j += NH) {              // eight results in flight, added in order
                    float v[NH][VEC];
#pragma unroll
                    for (int q = 0; q < NH; ++q)
#pragma unroll
                        for (int e = 0; e < VEC; ++e) v[q][e] = ONE && j == 0 ? h1[DEP ? q : 0][e] : hr[(size_t)min(j + q, A.hist_i - 1) * A.hist_stride + c + e];
#pragma unroll
                    for (int q = 0; q < NH; ++q)
                        if (j + q < A.hist_i) {
#pragma unroll
                            for (int e = 0; e < VEC; ++e) a[e] = __builtin_fmaf(A.dwa[j + q], v[q][e], a[e]);
                        }
                }
#pragma unroll
                for (int e = 0; e < VEC; ++e) r[e] = __builtin_fmaf(A.dwa[A.hist_i], r[e], a[e]);
            }
        }
        if (!A.rows) {
#pragma unroll
            for (int e = 0; e < VEC; ++e) xr[c + e] = r[e];
        }
        if (A.emb_save) {
#pragma unroll
            for (int e = 0; e < VEC; ++e) A.emb_save[(size_t)src * A.W + c + e] = r[e];
        }
#pragma unroll
        for (int e = 0; e < VEC; ++e) { sm[c + e] = r[e]; ss = __builtin_fmaf(r[e], r[e], ss); }
    }
    float rs = 1.f;
    if (A.w) rs = 1.0f / sqrtf(ob_block_sum(ss, red) / (float)A.W + A.eps);               // (uniform)
    E *out = (E *)A.out;
    for (int c = tid * VEC; c < A.W; c += stride) {
        ob_float4 v = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int e = 0; e < VEC; ++e) v[e] = A.w ? sm[c + e] * rs * (A.off + A.w[c + e]) : sm[c + e];
        if constexpr (VEC == 4) {
            const typename ObElem<E>::V4 o = ob_to_v4<E>(v);
            *reinterpret_cast<typename ObElem<E>::V4 *>(out + ob_frag<E>(t, c, A.out_nkt)) = o;
            if (A.out_rm) *reinterpret_cast<typename ObElem<E>::V4 *>((E *)A.out_rm + (size_t)t * A.ld_rm + c) = o;
        } else {
            out[ob_frag<E>(t, c, A.out_nkt)] = (E)v[0];
            if (A.out_rm) ((E *)A.out_rm)[(size_t)t * A.ld_rm + c] = (E)v[0];
        }
    }
}

// grid (norm groups, rows): v = y * silu(gate); out[k0 + i] = v / sqrt(mean over the group v^2 + eps) * w
struct ObGatedNormArgs {
    const void *y; int ldy; const void *gate; int ldg;       // row-major; the gate is the leading columns of the input product
    const float *w; float eps; int gsize;
    void *out; int out_nkt;
};
template <typename E, int VEC>                                 // VEC = 16 bytes of elements, or 1
__global__ __launch_bounds__(256) void ob_gated_norm_kernel(const ObGatedNormArgs A)
{
    typedef typename ObElem<E>::V16 V16;
    extern __shared__ __attribute__((aligned(16))) float sm[];
    float *red = sm + ((A.gsize + 3) & ~3);
    const int t = blockIdx.y, c0 = blockIdx.x * A.gsize, tid = threadIdx.x, stride = blockDim.x * VEC;
    const E *y = (const E *)A.y + (size_t)t * A.ldy + c0, *z = (const E *)A.gate + (size_t)t * A.ldg + c0;
    float ss = 0.f;
    for (int c = tid * VEC; c < A.gsize; c += stride) {
        V16 yv, zv;
        if constexpr (VEC > 1) { yv = *reinterpret_cast<const V16 *>(y + c); zv = *reinterpret_cast<const V16 *>(z + c); }
        else { yv[0] = y[c]; zv[0] = z[c]; }
#pragma unroll
        for (int e = 0; e < VEC; ++e) {
            const float v = (float)yv[e] * ob_silu<E>((float)zv[e]);
            sm[c + e] = v;
            ss = __builtin_fmaf(v, v, ss);
        }
    }
    ss = ob_block_sum(ss, red);
    const float rs = 1.0f / sqrtf(ss / (float)A.gsize + A.eps);
    E *out = (E *)A.out;
    for (int c = tid * VEC; c < A.gsize; c += stride) {
        V16 v;
#pragma unroll
        for (int e = 0; e < VEC; ++e) v[e] = (E)(sm[c + e] * rs * A.w[c0 + c + e]);
        if constexpr (VEC > 1) *reinterpret_cast<V16 *>(out + ob_frag<E>(t, c0 + c, A.out_nkt)) = v;       // (16 bytes of a row are contiguous)
        else out[ob_frag<E>(t, c0 + c, A.out_nkt)] = v[0];
    }
}

// greedy token: the smallest index of the largest logit of every row
__global__ __launch_bounds__(1024) void ob_argmax_rows_kernel(const float *__restrict__ logits, int32_t *__restrict__ next, int V)
{
    __shared__ float bv[16];
    __shared__ int bi[16];
    const float *l = logits + (size_t)blockIdx.x * V;
    const int tid = threadIdx.x;
    float best = -INFINITY;
    int idx = 0x7fffffff;
    if ((V & 3) == 0) {
        for (int i0 = tid; i0 < V / 4; i0 += 4096) {                  // four 16-byte loads in flight
            ob_float4 v[4];
#pragma unroll
            for (int j = 0; j < 4; ++j) v[j] = reinterpret_cast<const ob_float4 *>(l)[min(i0 + 1024 * j, V / 4 - 1)];
#pragma unroll
            for (int j = 0; j < 4; ++j)
#pragma unroll
                for (int e = 0; e < 4; ++e)                           // (ascending indices; a clamped repeat is not larger)
                    if (v[j][e] > best) { best = v[j][e]; idx = 4 * min(i0 + 1024 * j, V / 4 - 1) + e; }
        }
    } else {
        for (int i = tid; i < V; i += 1024) {
            const float v = l[i];
            if (v > best) { best = v; idx = i; }
        }
    }
#pragma unroll
    for (int s = 32; s > 0; s >>= 1) {
        const float ov = __shfl_xor(best, s);
        const int oi = __shfl_xor(idx, s);
        if (ov > best || (ov == best && oi < idx)) { best = ov; idx = oi; }
    }
    if ((tid & 63) == 0) { bv[tid >> 6] = best; bi[tid >> 6] = idx; }
    __syncthreads();
    if (tid == 0) {
        for (int w = 1; w < 16; ++w)
            if (bv[w] > best || (bv[w] == best && bi[w] < idx)) { best = bv[w]; idx = bi[w]; }
        next[blockIdx.x] = idx == 0x7fffffff ? 0 : idx;
    }
}
