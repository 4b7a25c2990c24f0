// Row kernels of the hybrid decoders: the residual stream in fp32 between the two matrix products of a layer, the gated group norm
// behind a recurrent mixer, and the greedy token.
#pragma once
#include "ob_dense.h"

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
            const float *zr = A.z + (size_t)src * A.ldz + c;
            for (int k = 0; k < A.n_split; k += 4) {                  // four splits in flight, added in order
                float zv[4][VEC];
#pragma unroll
                for (int j = 0; j < 4; ++j)
#pragma unroll
                    for (int e = 0; e < VEC; ++e) zv[j][e] = zr[(size_t)min(k + j, A.n_split - 1) * A.z_split + e];
#pragma unroll
                for (int j = 0; j < 4; ++j)
                    if (k + j < A.n_split) {
#pragma unroll
                        for (int e = 0; e < VEC; ++e) s[e] += zv[j][e];
                    }
            }
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
