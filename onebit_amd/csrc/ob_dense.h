// Dense matrix products of the hybrid decoders (bf16 MFMA with fp32 accumulation; the same kernels in true fp32) for gfx950.
//
// FRAGMENT-MAJOR operands: both the weights (packed once at load) and the activations (written that way by their producers) are
// stored as tiles of 16 rows x KT columns (KT = 32 bf16 / 16 fp32), 1 KB each, in the lane order of the MFMA operand: lane l holds
// row l & 15, columns (l >> 4) * EPL .. + EPL - 1 (EPL = 8 / 4, 16 bytes).  A tile is one contiguous 1 KB block, so
//   * a wave streams weights with perfectly linear 1 KB loads (decode: straight from HBM to the operand registers),
//   * LDS staging is a linear DMA and the operand read a linear ds_read_b128: no swizzle, no bank conflict, no address arithmetic,
//   * rows and columns are padded to whole tiles at load: the K loop has no masks for any model size.
// fp32: four v_mfma_f32_16x16x4_f32 per tile pair; element j of every lane's four is one instruction's k, the same on both operands.
// Products are computed transposed, D[n][t] = sum_k W[n][k] A[t][k]: a lane holds four consecutive output columns n of one token t.
#pragma once
#include "ob_common.h"

typedef __bf16 ob_bf8 __attribute__((ext_vector_type(8)));
typedef __bf16 ob_bf4 __attribute__((ext_vector_type(4)));

template <typename E> struct ObElem;
template <> struct ObElem<__bf16> {
    typedef ob_bf8 V16;                       // 16 bytes of operand
    typedef ob_bf4 V4;
    static constexpr int EPL = 8, KT = 32;
    static __device__ __forceinline__ ob_float4 mma(V16 a, V16 b, ob_float4 c) { return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0); }
};
template <> struct ObElem<float> {
    typedef ob_float4 V16;
    typedef ob_float4 V4;
    static constexpr int EPL = 4, KT = 16;
    static __device__ __forceinline__ ob_float4 mma(V16 a, V16 b, ob_float4 c)
    {
#pragma unroll
        for (int j = 0; j < 4; ++j) c = __builtin_amdgcn_mfma_f32_16x16x4f32(a[j], b[j], c, 0, 0, 0);
        return c;
    }
};

template <typename E> __device__ __forceinline__ typename ObElem<E>::V4 ob_to_v4(ob_float4 v)
{
    typename ObElem<E>::V4 o;
#pragma unroll
    for (int i = 0; i < 4; ++i) o[i] = (E)v[i];
    return o;
}
template <typename E> __device__ __forceinline__ ob_float4 ob_load4f(const E *p)
{
    const typename ObElem<E>::V4 v = *reinterpret_cast<const typename ObElem<E>::V4 *>(p);
    return (ob_float4){(float)v[0], (float)v[1], (float)v[2], (float)v[3]};
}

// two floats as bf16 pairs hi + lo: hi = the upper halves (truncated), lo = what is left, rounded -- 16 bits of mantissa together
typedef __bf16 ob_bf2 __attribute__((ext_vector_type(2)));
__device__ __forceinline__ uint32_t ob_pack_bf2(float a, float b) { return __builtin_bit_cast(uint32_t, __builtin_convertvector((ob_float2){a, b}, ob_bf2)); }
__device__ __forceinline__ void ob_split_bf2(float a, float b, uint32_t &hi, uint32_t &lo)
{
    const uint32_t ua = __float_as_uint(a), ub = __float_as_uint(b);
    hi = __builtin_amdgcn_perm(ub, ua, 0x07060302u);
    lo = ob_pack_bf2(a - __uint_as_float(ua & 0xffff0000u), b - __uint_as_float(ub & 0xffff0000u));
}

// element offset of (row, k) in a fragment-major matrix with nkt tiles per 16-row band
template <typename E> __host__ __device__ __forceinline__ size_t ob_frag(int row, int k, int nkt)
{
    constexpr int EPL = ObElem<E>::EPL, KT = ObElem<E>::KT;
    return ((size_t)(row >> 4) * nkt + k / KT) * (16 * KT) + (size_t)((k % KT) / EPL) * (16 * EPL) + (row & 15) * EPL + k % EPL;
}

__device__ __forceinline__ float ob_sigmoidf(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ __forceinline__ float ob_siluf(float z) { return z * ob_sigmoidf(z); }
// the 16-bit path's form: exp2 and reciprocal instructions, 1 ulp each in fp32
__device__ __forceinline__ float ob_silu_fast(float z) { return z * __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-1.4426950408889634f * z)); }
template <typename E> __device__ __forceinline__ float ob_silu(float z)
{
    if constexpr (sizeof(E) == 2) return ob_silu_fast(z); else return ob_siluf(z);
}
// tanh form of gelu; 0.5 (1 + tanh(u)) = sigmoid(2 u)
template <typename E> __device__ __forceinline__ float ob_gelu_tanh(float z)
{
    const float u = 0.79788456080286536f * (z + 0.044715f * z * z * z);
    if constexpr (sizeof(E) == 2) return z * __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-2.8853900817779268f * u));
    else return z * ob_sigmoidf(2.0f * u);
}
// quadratic above zero, exponential below, slope 1/2 at zero:  a z^2 + z / 2  |  b (e^z - 1 - z) + z / 2
template <typename E> __device__ __forceinline__ float ob_xielu(float z, float a, float b)
{
    const float n = fminf(z, 0.f);
    float em;
    if constexpr (sizeof(E) == 2) em = __builtin_amdgcn_exp2f(1.4426950408889634f * n) - 1.0f; else em = expm1f(n);
    return z > 0.f ? __builtin_fmaf(a * z, z, 0.5f * z) : __builtin_fmaf(b, em - n, 0.5f * z);
}
__device__ __forceinline__ float ob_softplusf(float z) { return fmaxf(z, 0.0f) + log1pf(expf(-fabsf(z))); }

// ---- what a product's output becomes -------------------------------------------------------------------------------------
//   OB_EPI_IN     the layer's input product [mixer columns | auxiliary fp32 columns | gate / up tile pairs]:
//                 mixer columns (+ bias) row-major u[t][n]; auxiliary columns fp32 aux[t][.]; act = silu(gate) * up into the
//                 fragment-major rows of the output product, at column act_k0
//   OB_EPI_PART   fp32 partial sums z[split][t][n] (the layer's output product: the row kernel that follows adds the splits)
//   OB_EPI_LOGITS fp32 logits[t][n], cap * tanh(v / cap) when cap > 0
//   OB_EPI_ACT    f(v) into fragment-major rows at column act_k0 + n: f = identity or xIELU
//   OB_EPI_HEADS  head-major rows: heads[n / D][t][n % D] (D a power of two), keys and values of a prompt's latents
//   OB_EPI_QFRAG  per token and 16 heads (columns n = head D + r) the operand tiles of a score product, heads as its rows: bf16
enum ObEpilogue { OB_EPI_IN = 0, OB_EPI_PART = 1, OB_EPI_LOGITS = 2, OB_EPI_ACT = 3, OB_EPI_HEADS = 4, OB_EPI_QFRAG = 5 };
enum ObDenseFn { OB_FN_ID = 0, OB_FN_XIELU = 1 };

// ---- which weights meet which rows ------------------------------------------------------------------------------------------
//   OB_ROWS_ALL     every row, fragment-major activations
//   OB_ROWS_HEADS   block-diagonal over heads: n tiles tile_group apart read their own act_cols columns of ROW-MAJOR activations
//   OB_ROWS_GATHER  blocks of one expert's rows (ObRowBlock table): activation row gather[row] of a ROW-MAJOR matrix, output row `row`
//   OB_ROWS_SORTED  the same blocks, fragment-major activations in block order
//   OB_ROWS_TABLE   few rows, formed here: gelu_tanh(sum of `n_pre` partial sums of another product) times the token's row of a table
//   OB_ROWS_SEGS    rows of several requests' cache slots (fragment-major bands), output rows consecutive per request
enum ObRowForm { OB_ROWS_ALL = 0, OB_ROWS_HEADS = 1, OB_ROWS_GATHER = 2, OB_ROWS_SORTED = 3, OB_ROWS_SEGS = 4, OB_ROWS_TABLE = 5 };
struct ObRowBlock { int32_t group, row0, count, pad; };      // rows [row0, row0 + count) of weight group `group`; row0 a multiple of 16 at a group's start

struct ObDenseArgs {
    const void *w, *a;             // fragment-major weights [n_tiles][nkt], activations [t tiles][nkt]
    int n_tiles, nkt, T;
    int kt_split;                  // k tiles per split (grid.y splits)
    // OB_EPI_IN
    const float *bias;             // [16 * nt_mix] or NULL
    void *u; int nt_mix;           // u: [T][16 * nt_mix]
    float *aux; int nt_aux;        // aux: [T][16 * nt_aux]; n tile nt_mix + nt_aux opens the gate / up pairs
    void *act; int act_k0, act_nkt;
    // OB_EPI_PART
    float *z; int ldz; size_t z_split;
    // OB_EPI_LOGITS
    float *logits; int V; float cap;
    // OB_EPI_ACT (act, act_k0, act_nkt as above)
    int fn; float fa, fb;          // xIELU's two factors
    // OB_EPI_HEADS, OB_EPI_QFRAG (D = 1 << d_shift; head_rows: rows per head / tiles of 16 heads)
    void *heads; int d_shift, head_rows;
    // OB_ROWS_HEADS / OB_ROWS_GATHER: row-major activations
    int lda, tile_group, act_cols;
    // OB_ROWS_TABLE: pre [n_pre][T][ld_pre] fp32, columns nkt KT
    const float *pre; int n_pre, ld_pre;
    const void *table; const int32_t *tokens; int ld_table, table_cols;      // entry (tokens[t], n), n < table_cols
    // OB_ROWS_GATHER / OB_ROWS_SORTED
    const ObRowBlock *blk; const int32_t *gather; size_t w_group;             // weight tiles per group
};
#define OB_DENSE_MAXSEG 64
struct ObDenseSegArgs : ObDenseArgs {          // OB_ROWS_SEGS: token block b belongs to segment i with blk_end[i - 1] <= b < blk_end[i]
    int nseg;
    int blk_end[OB_DENSE_MAXSEG];
    int band0[OB_DENSE_MAXSEG], row0[OB_DENSE_MAXSEG], rows[OB_DENSE_MAXSEG];
};

// (a class template, not an expression of the row form: kernel names must be the same on host and device)
template <int ROWS> struct ObDenseArgsOf { typedef ObDenseArgs type; };
template <> struct ObDenseArgsOf<OB_ROWS_SEGS> { typedef ObDenseSegArgs type; };

// one n-tile pair (nt even) of one token tile: lane = (token t, columns 16 nt + 4 g ..), (token t, columns 16 (nt + 1) + 4 g ..)
template <typename E, int EPI>
__device__ __forceinline__ void ob_dense_epilogue(const ObDenseArgs &A, int nt, int t, bool live, int g, ob_float4 v0, ob_float4 v1, int split)
{
    if (!live) return;
    if constexpr (EPI == OB_EPI_ACT || EPI == OB_EPI_HEADS || EPI == OB_EPI_QFRAG) {
#pragma unroll
        for (int h = 0; h < 2; ++h) {
            if (nt + h >= A.n_tiles) return;
            ob_float4 v = h ? v1 : v0;
            const int n = (nt + h) * 16 + 4 * g;
            if constexpr (EPI == OB_EPI_QFRAG) {
                const int hd = n >> A.d_shift, r = n & ((1 << A.d_shift) - 1);
                *reinterpret_cast<typename ObElem<E>::V4 *>((E *)A.heads + ((((size_t)t * A.head_rows + (hd >> 4)) << (A.d_shift + 4)) + ob_frag<E>(hd & 15, r, 0))) = ob_to_v4<E>(v);
            } else if constexpr (EPI == OB_EPI_HEADS) {
                const int hd = n >> A.d_shift, d = n & ((1 << A.d_shift) - 1);
                *reinterpret_cast<typename ObElem<E>::V4 *>((E *)A.heads + ((((size_t)hd * A.head_rows + t) << A.d_shift) + d)) = ob_to_v4<E>(v);
            } else {
                if (A.fn == OB_FN_XIELU) {
#pragma unroll
                    for (int e = 0; e < 4; ++e) v[e] = ob_xielu<E>(v[e], A.fa, A.fb);
                }
                *reinterpret_cast<typename ObElem<E>::V4 *>((E *)A.act + ob_frag<E>(t, A.act_k0 + n, A.act_nkt)) = ob_to_v4<E>(v);
            }
        }
    } else if constexpr (EPI == OB_EPI_PART) {
        float *z = A.z + (size_t)split * A.z_split + (size_t)t * A.ldz;
        if (nt < A.n_tiles) *reinterpret_cast<ob_float4 *>(z + nt * 16 + 4 * g) = v0;
        if (nt + 1 < A.n_tiles) *reinterpret_cast<ob_float4 *>(z + nt * 16 + 16 + 4 * g) = v1;
    } else if constexpr (EPI == OB_EPI_LOGITS) {
#pragma unroll
        for (int h = 0; h < 2; ++h) {
            ob_float4 v = h ? v1 : v0;
            const int n = (nt + h) * 16 + 4 * g;
            if (A.cap > 0.f) {
#pragma unroll
                for (int e = 0; e < 4; ++e) v[e] = A.cap * tanhf(v[e] / A.cap);
            }
            float *o = A.logits + (size_t)t * A.V + n;
            if ((A.V & 3) == 0) {
                if (n < A.V) *reinterpret_cast<ob_float4 *>(o) = v;
            } else {
                for (int e = 0; e < 4; ++e) if (n + e < A.V) o[e] = v[e];
            }
        }
    } else {
        if (nt >= A.n_tiles) return;
        const int n_plain = A.nt_mix + A.nt_aux;
        if (nt >= n_plain) {                            // (wave-uniform) gate tile, up tile
            ob_float4 o;
#pragma unroll
            for (int e = 0; e < 4; ++e) o[e] = ob_silu<E>(v0[e]) * v1[e];
            const int k = A.act_k0 + ((nt - n_plain) >> 1) * 16 + 4 * g;
            *reinterpret_cast<typename ObElem<E>::V4 *>((E *)A.act + ob_frag<E>(t, k, A.act_nkt)) = ob_to_v4<E>(o);
            return;
        }
#pragma unroll
        for (int h = 0; h < 2; ++h) {
            const int i = nt + h, n = i * 16 + 4 * g;
            ob_float4 v = h ? v1 : v0;
            if (i < A.nt_mix) {
                if (A.bias) v += *reinterpret_cast<const ob_float4 *>(A.bias + n);
                *reinterpret_cast<typename ObElem<E>::V4 *>((E *)A.u + (size_t)t * (16 * A.nt_mix) + n) = ob_to_v4<E>(v);
            } else if (i < n_plain) {
                *reinterpret_cast<ob_float4 *>(A.aux + (size_t)t * (16 * A.nt_aux) + (n - 16 * A.nt_mix)) = v;
            }
        }
    }
}

// four columns of a row of the OB_ROWS_TABLE operand
template <typename E> __device__ __forceinline__ void ob_table_piece(const ObDenseArgs &A, E *dst, int t, int n)
{
    const float *zp = A.pre + (size_t)t * A.ld_pre + n;
    const E *row = (const E *)A.table + (size_t)A.tokens[t] * A.ld_table + n;
    ob_float4 v = {0.f, 0.f, 0.f, 0.f}, tv = v;
    for (int k = 0; k < A.n_pre; k += 4) {                             // four splits in flight, added in order
        ob_float4 zv[4];
#pragma unroll
        for (int j = 0; j < 4; ++j) zv[j] = *reinterpret_cast<const ob_float4 *>(zp + (size_t)min(k + j, A.n_pre - 1) * A.T * A.ld_pre);
#pragma unroll
        for (int j = 0; j < 4; ++j) if (k + j < A.n_pre) v += zv[j];
    }
#pragma unroll
    for (int e = 0; e < 4; ++e) if (n + e < A.table_cols) tv[e] = (float)row[e];
#pragma unroll
    for (int e = 0; e < 4; ++e) v[e] = n + e < A.table_cols ? ob_gelu_tanh<E>(v[e]) * tv[e] : 0.f;
    *reinterpret_cast<typename ObElem<E>::V4 *>(dst + ob_frag<E>(t, n, A.nkt)) = ob_to_v4<E>(v);
}
// ... of many rows, in memory: grid (pieces / 256)
template <typename E> __global__ __launch_bounds__(256) void ob_table_rows_kernel(const ObDenseArgs A)
{
    const int nv = A.nkt * ObElem<E>::KT / 4;
    const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
    if (i < (int64_t)A.T * nv) ob_table_piece<E>(A, (E *)A.act, (int)(i / nv), 4 * (int)(i % nv));
}

// ---- few rows (T <= 64): weights from HBM straight into the operand registers ------------------------------------------
// Workgroup = 2 n tiles (32 output columns; a gate / up pair) x all token tiles x one K split; its four waves take a quarter of the
// split's k tiles each and add up through LDS.  Activations come from L2 (1 KB linear loads).  The next U k tiles are requested
// before the current U are multiplied: U * 2 KB of weights per wave in flight.
// Row-major activations (OB_ROWS_HEADS, OB_ROWS_GATHER): a lane's 16 bytes come from its own row, 64 bytes per row and k tile.
// Expert blocks: grid.z = entries of the block table (count 0: nothing to do).
template <typename E, int EPI, int MT, int ROWS = OB_ROWS_ALL>
__global__ __launch_bounds__(256, MT >= 4 ? 2 : 3) void ob_dense_skinny_kernel(const ObDenseArgs A)
{
    typedef typename ObElem<E>::V16 V16;
    constexpr int U = MT >= 4 ? 2 : 4;
    __shared__ ob_float4 red[4][2][MT][64];
    extern __shared__ __attribute__((aligned(16))) char formed[];      // OB_ROWS_TABLE: [MT][nkt] tiles
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int nt = blockIdx.x * 2, split = blockIdx.y;
    const int k_lo = split * A.kt_split, k_hi = min(A.nkt, k_lo + A.kt_split);
    const int per = (k_hi - k_lo + 3) >> 2;
    const int k0 = k_lo + wave * per, k1 = min(k0 + per, k_hi);
    int t0 = 0, rows = A.T;
    size_t wg = 0;
    if constexpr (ROWS == OB_ROWS_GATHER || ROWS == OB_ROWS_SORTED) {
        const ObRowBlock b = A.blk[blockIdx.z];
        if (b.count <= 0) return;                        // (uniform)
        t0 = b.row0; rows = b.count; wg = (size_t)b.group * A.w_group;
    }
    const V16 *w0 = (const V16 *)A.w + (wg + (size_t)nt * A.nkt) * 64 + lane;
    const V16 *w1 = (const V16 *)A.w + (wg + (size_t)min(nt + 1, A.n_tiles - 1) * A.nkt) * 64 + lane;
    if constexpr (ROWS == OB_ROWS_TABLE) {
        const int nv = A.nkt * ObElem<E>::KT / 4;
        for (int i = tid; i < A.T * nv; i += 256) ob_table_piece<E>(A, (E *)formed, i / nv, 4 * (i % nv));
        __syncthreads();
    }
    // this lane's piece of k tile 0 of every token tile, and the step (in 16 bytes) to the next k tile
    const V16 *ap[MT];
    constexpr int KSTEP = ROWS == OB_ROWS_HEADS || ROWS == OB_ROWS_GATHER ? 4 : 64;
#pragma unroll
    for (int m = 0; m < MT; ++m) {
        if constexpr (ROWS == OB_ROWS_HEADS)
            ap[m] = (const V16 *)((const E *)A.a + (size_t)min(m * 16 + (lane & 15), rows - 1) * A.lda + nt / A.tile_group * A.act_cols) + (lane >> 4);
        else if constexpr (ROWS == OB_ROWS_GATHER)
            ap[m] = (const V16 *)((const E *)A.a + (size_t)A.gather[t0 + min(m * 16 + (lane & 15), rows - 1)] * A.lda) + (lane >> 4);
        else if constexpr (ROWS == OB_ROWS_TABLE) ap[m] = (const V16 *)formed + lane + (size_t)m * A.nkt * 64;
        else ap[m] = (const V16 *)A.a + lane + (size_t)((t0 >> 4) + m) * A.nkt * 64;
    }
    ob_float4 acc[2][MT];
#pragma unroll
    for (int m = 0; m < MT; ++m) acc[0][m] = acc[1][m] = (ob_float4){0.f, 0.f, 0.f, 0.f};
    V16 wc[2][U], ac[MT][U], wn[2][U], an[MT][U];
    auto fetch = [&](V16 (&wd)[2][U], V16 (&ad)[MT][U], int k) {
#pragma unroll
        for (int u = 0; u < U; ++u) {
            const int kk = min(k + u, k1 - 1);
            wd[0][u] = __builtin_nontemporal_load(w0 + (size_t)kk * 64);
            wd[1][u] = __builtin_nontemporal_load(w1 + (size_t)kk * 64);
#pragma unroll
            for (int m = 0; m < MT; ++m) ad[m][u] = ap[m][(size_t)kk * KSTEP];
        }
    };
    if (k0 < k1) {                                       // (wave-uniform)
        fetch(wc, ac, k0);
        for (int k = k0; k < k1; k += U) {
            const bool more = k + U < k1;
            if (more) fetch(wn, an, k + U);
#pragma unroll
            for (int u = 0; u < U; ++u) {
                if (k + u < k1) {
#pragma unroll
                    for (int m = 0; m < MT; ++m) {
                        acc[0][m] = ObElem<E>::mma(wc[0][u], ac[m][u], acc[0][m]);
                        acc[1][m] = ObElem<E>::mma(wc[1][u], ac[m][u], acc[1][m]);
                    }
                }
            }
            if (more) {
#pragma unroll
                for (int u = 0; u < U; ++u) {
                    wc[0][u] = wn[0][u]; wc[1][u] = wn[1][u];
#pragma unroll
                    for (int m = 0; m < MT; ++m) ac[m][u] = an[m][u];
                }
            }
        }
    }
#pragma unroll
    for (int h = 0; h < 2; ++h)
#pragma unroll
        for (int m = 0; m < MT; ++m) red[wave][h][m][lane] = acc[h][m];
    __syncthreads();
    for (int m = wave; m < MT; m += 4) {
        ob_float4 v[2];
#pragma unroll
        for (int h = 0; h < 2; ++h) v[h] = (red[0][h][m][lane] + red[1][h][m][lane]) + (red[2][h][m][lane] + red[3][h][m][lane]);
        const int tl = m * 16 + (lane & 15);
        ob_dense_epilogue<E, EPI>(A, nt, t0 + tl, tl < rows, lane >> 4, v[0], v[1], split);
    }
}

// ---- many rows: LDS-DMA tiles ------------------------------------------------------------------------------------------
// Workgroup = NB n tiles x TB token tiles, waves WN x WT; NST stages of one k tile each in LDS, filled by 1 KB DMAs, ONE raw barrier
// per k tile behind a counted vmcnt: at the top of step k the tile k has landed (at most the NST - 2 younger ones are outstanding),
// the barrier tells everyone, and the buffer of tile k - 1 -- whose operand reads are complete -- takes tile k + NST - 1.
__device__ __forceinline__ void ob_dma_1k(const char *base, uint32_t lane_off, uint32_t lds_addr)
{
    uint32_t keep;
    asm volatile("s_mov_b32 %0, m0\n\ts_mov_b32 m0, %1\n\ts_nop 0\n\tglobal_load_lds_dwordx4 %2, %3\n\ts_mov_b32 m0, %0"
                 : "=&s"(keep) : "s"(lds_addr), "v"(lane_off), "s"(base) : "memory");
}

template <typename E, int EPI, int NB, int TB, int WN, int WT, int NST, int ROWS = OB_ROWS_ALL>
__global__ __launch_bounds__(64 * WN * WT, 2) void ob_dense_tile_kernel(const typename ObDenseArgsOf<ROWS>::type A)
{
    static_assert(ROWS != OB_ROWS_HEADS, "the block-diagonal form has few rows only");
    typedef typename ObElem<E>::V16 V16;
    constexpr int NW = WN * WT, TILES = NB + TB, PER = TILES / NW, MN = NB / WN, MT = TB / WT;
    static_assert(TILES % NW == 0 && NB % WN == 0 && TB % WT == 0 && MN % 2 == 0, "tile shape");
    extern __shared__ __attribute__((aligned(16))) char smem[];
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int wn = wave % WN, wt = wave / WN;
    // XCD-aware numbering: workgroup ids are dealt round-robin to the 8 XCDs; give each a contiguous range of logical tiles, token
    // blocks fastest, so that the tiles in flight on an XCD share weight bands and activation rows in its L2
    const int ntb = (A.T + TB * 16 - 1) / (TB * 16);                   // (grouped forms: T = 16 TB times the number of blocks)
    const int nwg = gridDim.x, orig = blockIdx.x, xcd = orig & 7, q8 = nwg >> 3, rem = nwg & 7;
    const int bid = (xcd < rem ? xcd * (q8 + 1) : rem * (q8 + 1) + (xcd - rem) * q8) + (orig >> 3);
    const int nb = bid / ntb, tb = bid - nb * ntb;
    const int n0 = nb * NB, split = blockIdx.y;
    // rows of this block: `rows` of them, activations from band `band0` on, outputs from row `out0` on
    int band0 = tb * TB, out0 = tb * TB * 16, rows = A.T - out0;
    size_t wg = 0;
    if constexpr (ROWS == OB_ROWS_GATHER || ROWS == OB_ROWS_SORTED) {
        const ObRowBlock b = A.blk[tb];
        if (b.count <= 0) return;                                     // (uniform)
        band0 = b.row0 >> 4; out0 = b.row0; rows = b.count; wg = (size_t)b.group * A.w_group;
    } else if constexpr (ROWS == OB_ROWS_SEGS) {
        int sg = 0;
        while (sg < A.nseg - 1 && tb >= A.blk_end[sg]) ++sg;
        const int loc = (tb - (sg ? A.blk_end[sg - 1] : 0)) * TB;
        band0 = A.band0[sg] + loc; out0 = A.row0[sg] + loc * 16; rows = A.rows[sg] - loc * 16;
    }
    const int k_lo = split * A.kt_split, k_hi = min(A.nkt, k_lo + A.kt_split), nk = k_hi - k_lo;
    const int t_tiles = (rows + 15) >> 4;
    const char *src[PER];
    uint32_t loff[PER], kstep[PER];                                   // (two values, wave-uniform step: 1 KB tiles, or 64 bytes of a gathered row)
#pragma unroll
    for (int i = 0; i < PER; ++i) {
        const int j = wave * PER + i;
        const size_t band = j < NB ? (size_t)min(n0 + j, A.n_tiles - 1) : (size_t)(band0 + min(j - NB, t_tiles - 1));
        src[i] = (const char *)(j < NB ? A.w : A.a) + ((j < NB ? wg : 0) + band * A.nkt + k_lo) * 1024;
        loff[i] = lane * 16;
        kstep[i] = 1024;
        if constexpr (ROWS == OB_ROWS_GATHER) {
            if (j >= NB) {
                src[i] = (const char *)A.a + (size_t)k_lo * 64;
                loff[i] = (uint32_t)A.gather[out0 + min((j - NB) * 16 + (lane & 15), rows - 1)] * (uint32_t)(A.lda * sizeof(E)) + (lane >> 4) * 16;
                kstep[i] = 64;
            }
        }
    }
    const uint32_t lds0 = (uint32_t)(size_t)(__attribute__((address_space(3))) char *)smem;
    auto dma = [&](int k, int buf) {
        const size_t kk = (size_t)min(k, nk - 1);
#pragma unroll
        for (int i = 0; i < PER; ++i)
            ob_dma_1k(src[i] + kk * (ROWS == OB_ROWS_GATHER ? kstep[i] : 1024), ROWS == OB_ROWS_GATHER ? loff[i] : lane * 16,
                      lds0 + (uint32_t)(buf * TILES + wave * PER + i) * 1024);
    };
    ob_float4 acc[MN][MT];
#pragma unroll
    for (int i = 0; i < MN; ++i)
#pragma unroll
        for (int j = 0; j < MT; ++j) acc[i][j] = (ob_float4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int s = 0; s < NST - 1; ++s) dma(s, s);
    int buf = 0;
    for (int k = 0; k < nk; ++k) {
        asm volatile("s_waitcnt vmcnt(%0) lgkmcnt(0)\n\ts_barrier" :: "n"((NST - 2) * PER) : "memory");
        dma(k + NST - 1, buf == 0 ? NST - 1 : buf - 1);               // (past the end: the last tile again, into a buffer nobody reads)
        const V16 *base = reinterpret_cast<const V16 *>(smem + (size_t)buf * TILES * 1024) + lane;
        V16 wf[MN], af[MT];
#pragma unroll
        for (int j = 0; j < MT; ++j) af[j] = base[(NB + wt * MT + j) * 64];
#pragma unroll
        for (int i = 0; i < MN; ++i) wf[i] = base[(wn * MN + i) * 64];
        __builtin_amdgcn_s_setprio(1);
#pragma unroll
        for (int i = 0; i < MN; ++i)
#pragma unroll
            for (int j = 0; j < MT; ++j) acc[i][j] = ObElem<E>::mma(wf[i], af[j], acc[i][j]);
        __builtin_amdgcn_s_setprio(0);
        buf = buf + 1 == NST ? 0 : buf + 1;
    }
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");                  // no transfer may land after the workgroup's LDS is released
    const int g = lane >> 4;
#pragma unroll
    for (int j = 0; j < MT; ++j) {
        const int tl = (wt * MT + j) * 16 + (lane & 15);
#pragma unroll
        for (int i = 0; i < MN; i += 2) ob_dense_epilogue<E, EPI>(A, n0 + wn * MN + i, out0 + tl, tl < rows, g, acc[i][j], acc[i + 1][j], split);
    }
}
