// Latent attention: keys and values of all heads are projections of ONE small normalised vector c per token, and only c is cached.
//   c_q = rms(W_dq h) wq,  q = W_uq c_q;   c = rms(W_dkv h) wc;   k = W_uk c, v = W_uv c per head;   softmax(q.k scale) v over j <= i
// Two equal forms:
//   absorbed   q'_h = W_uk_h^T q_h (per head, kv_rank wide): the score is q'_h . c, the output W_uv_h (sum of weights times c) -- all heads
//              share one key row, which is its own value row.  Decoding, and whatever the tiled forms do not take.
//   expanded   k, v of a prompt's keys once (one product over the cache), then the flash kernel of ob_flash.h (ObFlSoftmaxBf16).
// Cache: fragment-major (ob_dense.h) [slots][max_len / 16][rp / KT] tiles, rp = kv_rank rounded up, columns beyond kv_rank zero: a band of 16
// keys IS the MFMA operand of a score product and the activation operand of the expansion.
#pragma once
#include "ob_dense.h"
#include "ob_flash.h"
#include "ob_hrows.h"

// ---- rows of the input product [W_dq | W_dkv] -> both norms; c_q to the fragment-major rows of the query product, c to the cache.  grid (rows).
struct ObLatPrepArgs {
    const float *z; size_t z_split; int n_split, ldz;
    int q_rank, c0, kv_rank;                   // c: columns c0 .. c0 + kv_rank of the product
    const float *qn_w, *kvn_w; float eps;
    void *cq; int cq_nkt;
    void *cache; int rp, bands;                // bands of 16 keys per slot
    const int32_t *row_slot, *row_pos; int n_slots, max_len;
};
template <typename E, int VEC>                                 // VEC 4: both ranks are multiples of 4
__global__ __launch_bounds__(1024) void ob_lat_prep_kernel(const ObLatPrepArgs A)
{
    constexpr int KT = ObElem<E>::KT;
    extern __shared__ __attribute__((aligned(16))) float sm[];        // [q_rank + kv_rank] | [16] reductions
    const int t = blockIdx.x, tid = threadIdx.x, stride = blockDim.x * VEC, n = A.q_rank + A.kv_rank;
    float *red = sm + ((n + 3) & ~3);
    const int slot = A.row_slot[t], pos = A.row_pos[t];
    const float *zr = A.z + (size_t)t * A.ldz;
    float sq = 0.f, sc = 0.f;
    for (int i = tid * VEC; i < n; i += stride) {
        float v[VEC];
#pragma unroll
        for (int e = 0; e < VEC; ++e) v[e] = 0.f;
        ob_sum_splits<VEC>(v, zr + (i < A.q_rank ? i : A.c0 + i - A.q_rank), A.z_split, A.n_split);
        float s = 0.f;
#pragma unroll
        for (int e = 0; e < VEC; ++e) { sm[i + e] = v[e]; s = __builtin_fmaf(v[e], v[e], s); }
        if (i < A.q_rank) sq += s; else sc += s;
    }
    sq = ob_block_sum(sq, red);
    sc = ob_block_sum(sc, red);
    const float rq = 1.0f / sqrtf(sq / (float)A.q_rank + A.eps), rc = 1.0f / sqrtf(sc / (float)A.kv_rank + A.eps);
    // c_q, then c: columns padded with zeros
    auto put = [&](E *dst, int row, int nkt, int cols, const float *src, const float *w, float r) {
        for (int i = tid * VEC; i < nkt * KT; i += stride) {
            ob_float4 v = {0.f, 0.f, 0.f, 0.f};
            if (i < cols) {
#pragma unroll
                for (int e = 0; e < VEC; ++e) v[e] = src[i + e] * r * w[i + e];
            }
            if constexpr (VEC == 4) *reinterpret_cast<typename ObElem<E>::V4 *>(dst + ob_frag<E>(row, i, nkt)) = ob_to_v4<E>(v);
            else dst[ob_frag<E>(row, i, nkt)] = (E)v[0];
        }
    };
    put((E *)A.cq, t, A.cq_nkt, A.q_rank, sm, A.qn_w, rq);
    if (slot < 0 || slot >= A.n_slots || pos < 0 || pos >= A.max_len) return;          // idle row
    const int nkt = A.rp / KT;
    put((E *)A.cache + (size_t)slot * A.bands * nkt * (16 * KT), pos, nkt, A.kv_rank, sm + A.q_rank, A.kvn_w, rc);
}

// ---- absorbed attention, any element type and size: one workgroup per (head, row), fp32 arithmetic with the accurate functions
struct ObLatArgs {
    const void *q; void *ctx; int ldq;         // ctx: rows [H][rp]; q too, or (decode form) per row and 16 heads the operand tiles of the score product
    const void *cache; int rp, bands;
    const int32_t *row_slot, *row_pos;
    int row0, H, n_slots, max_len;
    float scale;
    // decode form
    int chunk, nsplit;
    void *part; float *ml;                     // [rows][nsplit][H][rp] each split's own output, [rows][nsplit][H][2] its maximum (base 2) and sum
};
template <typename E>
__global__ __launch_bounds__(256) void ob_lat_rows_kernel(const ObLatArgs A)
{
    typedef typename ObElem<E>::V16 V16;
    constexpr int EPL = ObElem<E>::EPL, KT = ObElem<E>::KT;
    extern __shared__ __attribute__((aligned(16))) float qs[];        // [rp] query | [256] weights | [16] reductions
    float *ws = qs + A.rp, *red = ws + 256;
    const int h = blockIdx.x, row = A.row0 + blockIdx.y, tid = threadIdx.x, nkt = A.rp / KT;
    const int slot = A.row_slot[row], pos = A.row_pos[row];
    if (slot < 0 || slot >= A.n_slots || pos < 0 || pos >= A.max_len) return;
    const E *q = (const E *)A.q + (size_t)row * A.ldq + h * A.rp;
    E *o = (E *)A.ctx + (size_t)row * A.ldq + h * A.rp;
    const E *c = (const E *)A.cache + (size_t)slot * A.bands * nkt * (16 * KT);
    for (int d = tid; d < A.rp; d += 256) qs[d] = (float)q[d] * A.scale;
    for (int d0 = 0; d0 < A.rp; d0 += 256) {                          // (one pass up to 256 latent columns)
        const int d = d0 + tid;
        float acc = 0.f, m = -INFINITY, l = 0.f;
        for (int j0 = 0; j0 <= pos; j0 += 256) {
            __syncthreads();
            const int j = j0 + tid;
            float s = -INFINITY;
            if (j <= pos) {
                s = 0.f;
                for (int e = 0; e < A.rp; e += EPL) {
                    const V16 k = *reinterpret_cast<const V16 *>(c + ob_frag<E>(j, e, nkt));
#pragma unroll
                    for (int i = 0; i < EPL; ++i) s = __builtin_fmaf((float)k[i], qs[e + i], s);
                }
            }
            float mx = ob_wave_max(s);
            if ((tid & 63) == 0) red[tid >> 6] = mx;
            __syncthreads();
            mx = fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3]));
            const float mn = fmaxf(m, mx), keep = expf(m - mn);       // (j0 <= pos: the block has a visible key, mn is finite)
            const float w = j <= pos ? expf(s - mn) : 0.f;
            ws[tid] = w;
            l = l * keep + ob_block_sum(w, red + 4);                  // (its barriers also publish ws)
            m = mn;
            acc *= keep;
            if (d < A.rp) {
                const int nj = min(256, pos + 1 - j0);
                for (int jj = 0; jj < nj; ++jj) acc = __builtin_fmaf(ws[jj], (float)c[ob_frag<E>(j0 + jj, d, nkt)], acc);
            }
        }
        if (d < A.rp) o[d] = (E)(acc / l);
    }
}

// ---- absorbed attention, bf16 MFMA: one row, 16 HT heads, one key block ("split") of the context per workgroup; RP latent columns.
// Blocks of 64 keys, double-buffered in LDS (a band of 16 keys x 32 columns = one 1 KB tile) behind two more blocks on their way in registers:
// at 64 KB a block that is what keeps HBM busy at one workgroup per CU.  Four waves per tile of 16 heads: each scores
// one band (S^T = C . Q'^T, queries in registers); the scores pass through LDS once; every wave forms the weights of all 64 keys for its
// heads and multiplies them into its quarter of the latent columns (O^T = C^T . P^T, the SAME tiles through the transposing LDS read).
// Weights enter as two bf16 terms (16 bits of mantissa).  A tile's 16-byte pieces lie at [column group][row ^ (12 if the group is odd)]:
// both reads are free of bank conflicts.
template <int RP, int HT>
__global__ __launch_bounds__(256 * HT, RP >= 512 && HT == 1 ? 1 : 2) void ob_lat_dec_kernel(const ObLatArgs A)
{
    constexpr int NKT = RP / 32, DT = RP / 64;                        // k tiles of a score; 16-column output tiles per wave
    constexpr int STAGE = 4 * NKT * 1024, SLD = 68;
    typedef short ob_v4s __attribute__((ext_vector_type(4)));
    typedef short ob_v8s __attribute__((ext_vector_type(8)));
    typedef __attribute__((address_space(3))) ob_v4s ob_lds_v4s;
    extern __shared__ __attribute__((aligned(16))) char lsm[];        // two stages | scores [16 HT][SLD]
    const int tid = threadIdx.x, lane = tid & 63, wv = __builtin_amdgcn_readfirstlane(tid >> 6), wave = wv & 3, ht = wv >> 2, lr = lane & 15, g = lane >> 4;
    float *ss = reinterpret_cast<float *>(lsm + 2 * STAGE) + (16 * ht + lr) * SLD;     // this lane's head
    const int row = A.row0 + blockIdx.y, split = blockIdx.z, h = blockIdx.x * 16 * HT + 16 * ht + lr;
    ob_bf8 q[NKT];
    const ob_bf8 *qr = (const ob_bf8 *)A.q + ((size_t)row * ((A.H + 15) >> 4) + blockIdx.x * HT + ht) * NKT * 64 + lane;
#pragma unroll
    for (int k = 0; k < NKT; ++k) q[k] = qr[k * 64];                  // (a head beyond the last one: whatever is there, its output is not written)
    const int slot = __builtin_amdgcn_readfirstlane(A.row_slot[row]), pos = __builtin_amdgcn_readfirstlane(A.row_pos[row]);
    if (slot < 0 || slot >= A.n_slots || pos < 0 || pos >= A.max_len) return;          // idle row (uniform)
    const int L = pos + 1, p_lo = split * A.chunk;
    if (p_lo >= L) return;                                                             // empty split (uniform)
    const int p_hi = min(L, p_lo + A.chunk), nlive = (L + A.chunk - 1) / A.chunk, nb = (p_hi - p_lo + 63) >> 6, last_band = (L - 1) >> 4;
    const char *cs = (const char *)A.cache + (size_t)slot * A.bands * NKT * 1024;
    const uint32_t swz = (uint32_t)(16 * g + (lr ^ ((g & 1) ? 12 : 0))) * 16;          // this lane's piece of a tile in LDS
    constexpr int NP = NKT / HT;                                      // the waves of a band share its tiles
    ob_u32x4 on_way[2][NP];
    auto fetch = [&](ob_u32x4 (&r)[NP], int blk) {                    // (bands past the last key: the last one again)
        const ob_u32x4 *src = (const ob_u32x4 *)(cs + ((size_t)min((p_lo >> 4) + 4 * blk + wave, last_band) * NKT + ht * NP) * 1024) + lane;
#pragma unroll
        for (int i = 0; i < NP; ++i) r[i] = __builtin_nontemporal_load(src + i * 64);
    };
    auto put = [&](const ob_u32x4 (&r)[NP], int buf) {
        char *dst = lsm + buf * STAGE + (wave * NKT + ht * NP) * 1024 + swz;
#pragma unroll
        for (int i = 0; i < NP; ++i) *reinterpret_cast<ob_u32x4 *>(dst + i * 1024) = r[i];
    };
    fetch(on_way[0], 0);
    if (nb > 1) fetch(on_way[1], 1);
    ob_float4 acc[DT];
#pragma unroll
    for (int d = 0; d < DT; ++d) acc[d] = (ob_float4){0.f, 0.f, 0.f, 0.f};
    float m = -INFINITY, l = 0.f;
    const float sl = A.scale * 1.4426950408889634f;
    // transposing read of 16 columns from d0 on: lane i of a 16-lane group brings row 4 g + (i >> 2), columns d0 + 4 (i & 3) .. + 3
    const int vrow = 4 * g + (lr >> 2), vc = (lr & 3) >> 1;
    const uint32_t voff = (uint32_t)((vc * 16 + (vrow ^ (vc ? 12 : 0))) * 16 + (lr & 1) * 8);      // (column groups 2 j + vc: odd exactly when vc is)
    auto block = [&](const int b, auto odd) {
        constexpr int buf = decltype(odd)::value;
        put(on_way[buf], buf);                                        // (its last readers passed the barriers of block b - 1)
        if (b + 2 < nb) fetch(on_way[buf], b + 2);
        asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory");                // (no wait for what is on its way)
        const char *base = lsm + buf * STAGE;
        ob_float4 s[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};                 // (two chains)
#pragma unroll
        for (int k = 0; k < NKT; ++k) s[k & 1] = ObElem<__bf16>::mma(*reinterpret_cast<const ob_bf8 *>(base + (wave * NKT + k) * 1024 + swz), q[k], s[k & 1]);
        const int key = p_lo + 64 * b + 16 * wave + 4 * g;
        ob_float4 sc = (s[0] + s[1]) * sl;
#pragma unroll
        for (int e = 0; e < 4; ++e) if (key + e >= p_hi) sc[e] = -INFINITY;
        *reinterpret_cast<ob_float4 *>(ss + 16 * wave + 4 * g) = sc;
        asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory");
        ob_u32x4 wh[2], wl[2];
        ob_float4 w[4];
        float mx = -INFINITY;
#pragma unroll
        for (int k = 0; k < 4; ++k) {
            w[k] = *reinterpret_cast<const ob_float4 *>(ss + 16 * k + 4 * g);
#pragma unroll
            for (int e = 0; e < 4; ++e) mx = fmaxf(mx, w[k][e]);
        }
        mx = ob_fl_col_max(mx);                                       // (a block has at least one key: finite)
        if (__builtin_amdgcn_ballot_w64(mx - m > 8.0f) != 0) {        // the running maximum moves only when it must (-inf before the first block)
            const float mn = fmaxf(m, mx), keep = __builtin_amdgcn_exp2f(m - mn);
            l *= keep;
#pragma unroll
            for (int d = 0; d < DT; ++d) acc[d] *= keep;
            m = mn;
        }
#pragma unroll
        for (int k = 0; k < 4; ++k)
#pragma unroll
            for (int e = 0; e < 4; e += 2) {
                const float w0 = __builtin_amdgcn_exp2f(w[k][e] - m), w1 = __builtin_amdgcn_exp2f(w[k][e + 1] - m);
                l += w0 + w1;
                uint32_t hi, lo;
                ob_split_bf2(w0, w1, hi, lo);
                wh[k >> 1][2 * (k & 1) + (e >> 1)] = hi;
                wl[k >> 1][2 * (k & 1) + (e >> 1)] = lo;
            }
#pragma unroll
        for (int d = 0; d < DT; ++d) {
            const int dt = wave * DT + d;                             // columns 16 dt ..
            const char *vt = base + (dt >> 1) * 1024 + (dt & 1) * 512 + voff;
#pragma unroll
            for (int ks = 0; ks < 2; ++ks) {
                const ob_v4s lo = __builtin_amdgcn_ds_read_tr16_b64_v4i16((ob_lds_v4s *)(vt + 2 * ks * NKT * 1024));
                const ob_v4s hi = __builtin_amdgcn_ds_read_tr16_b64_v4i16((ob_lds_v4s *)(vt + (2 * ks + 1) * NKT * 1024));
                const ob_v8s a8 = {lo[0], lo[1], lo[2], lo[3], hi[0], hi[1], hi[2], hi[3]};
                const ob_bf8 a = __builtin_bit_cast(ob_bf8, a8);
                acc[d] = ObElem<__bf16>::mma(a, __builtin_bit_cast(ob_bf8, wh[ks]), acc[d]);
                acc[d] = ObElem<__bf16>::mma(a, __builtin_bit_cast(ob_bf8, wl[ks]), acc[d]);
            }
        }
    };
    for (int b = 0; b < nb; b += 2) {
        block(b, std::integral_constant<int, 0>());
        if (b + 1 < nb) block(b + 1, std::integral_constant<int, 1>());
    }
    // lane: head h, columns 16 dt + 4 g ..
    const float lt = ob_fl_col_sum(l);
    if (h >= A.H) return;
    const float inv = 1.0f / lt;
    const size_t at = ((size_t)row * A.nsplit + split) * A.H + h;
    __bf16 *o = (nlive == 1 ? (__bf16 *)A.ctx + (size_t)row * A.ldq + (size_t)h * RP : (__bf16 *)A.part + at * RP) + 16 * wave * DT + 4 * g;
#pragma unroll
    for (int d = 0; d < DT; ++d) *reinterpret_cast<ob_bf4 *>(o + 16 * d) = ob_to_v4<__bf16>(acc[d] * inv);
    if (nlive > 1 && wave == 0 && g == 0) { A.ml[2 * at] = m; A.ml[2 * at + 1] = lt; }
}

// ---- the splits of a context together: grid (heads, rows), rp / 8 threads rounded up to a wave
__global__ __launch_bounds__(256) void ob_lat_combine_kernel(const ObLatArgs A)
{
    const int h = blockIdx.x, row = A.row0 + blockIdx.y;
    const int slot = A.row_slot[row], pos = A.row_pos[row];
    if (slot < 0 || slot >= A.n_slots || pos < 0 || pos >= A.max_len) return;
    const int nlive = (pos + A.chunk) / A.chunk;
    if (nlive == 1) return;                                           // (written by the attention itself)
    const size_t at = (size_t)row * A.nsplit * A.H + h;
    // (at most 64 splits: lane s has split s)
    const int lane = threadIdx.x & 63;
    const float *pm = A.ml + 2 * (at + (size_t)min(lane, nlive - 1) * A.H);
    const float ms = lane < nlive ? pm[0] : -INFINITY, mx = ob_wave_max(ms);            // (whole wave)
    const float w = lane < nlive ? pm[1] * __builtin_amdgcn_exp2f(ms - mx) : 0.f;
    __shared__ float share[64];                                       // each split's share of the row's weight
    const float total = ob_wave_sum(w);
    if (threadIdx.x < 64) share[lane] = w / total;
    __syncthreads();
    const __bf16 *part = (const __bf16 *)A.part + at * A.rp;
    for (int d = threadIdx.x * 8; d < A.rp; d += blockDim.x * 8) {
        float o[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
        for (int s0 = 0; s0 < nlive; s0 += 8) {                       // eight splits in flight, added in order
            ob_bf8 v[8];
#pragma unroll
            for (int j = 0; j < 8; ++j) v[j] = *reinterpret_cast<const ob_bf8 *>(part + (size_t)min(s0 + j, nlive - 1) * A.H * A.rp + d);
#pragma unroll
            for (int j = 0; j < 8; ++j) {
                if (s0 + j >= nlive) break;
                const float f = share[s0 + j];
#pragma unroll
                for (int e = 0; e < 8; ++e) o[e] = __builtin_fmaf(f, (float)v[j][e], o[e]);
            }
        }
        ob_bf8 r;
#pragma unroll
        for (int e = 0; e < 8; ++e) r[e] = (__bf16)o[e];
        *reinterpret_cast<ob_bf8 *>((__bf16 *)A.ctx + (size_t)row * A.ldq + (size_t)h * A.rp + d) = r;
    }
}
