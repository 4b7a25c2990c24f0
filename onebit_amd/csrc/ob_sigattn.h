// Attention whose weights are sigmoids (not normalised over the keys) of scaled unit-RMS dot products minus a distance bias:
//   w(i, j) = sigmoid(rms(q_i) . rms(k_j) * scale - r1 ln(1 + r2 (i - j)) + pb),   o_i = sum_{j <= i} w(i, j) v_j
// r1, r2, pb per query head (r1 / pb may be NULL: no such term).  Partial results over disjoint key sets simply ADD, so a split
// context needs neither running maxima nor sums.  Weights are formed in fp32 in the base-2 domain: w = 1 / (1 + 2^a),
//   a = -scale log2(e) q.k + r1 log2(1 + r2 d) - pb log2(e)        (log2(e) ln(x) = log2(x)).
// Forms: ob_sig_prep_kernel (unit-RMS queries, keys; cache append) + the flash kernel of ob_flash.h with ObFlSigmoidBf16 (prompt rows,
// head sizes up to 128); ob_sig_dec_kernel (one new token per row, any context, everything fused); ob_sig_rows_kernel (any element
// type and head size, plain fp32 arithmetic).
// Cache: k [slots][G][max_len][kp], v [slots][G][max_len][vp], keys stored unit-RMS, columns beyond the head size zero.
#pragma once
#include "ob_dense.h"

struct ObSigBias { const float *r1, *r2, *pb; };
#define OB_LOG2E 1.4426950408889634f

// ---- prompt rows: unit-RMS q -> qn [T][H][kp]; k, v -> cache.  One wave per (row, head of q | k | v).
struct ObSigPrepArgs {
    const void *u; int ldu, row0;              // [q: H dim | k: G dim | v: G vdim] rows of the input product
    void *qn, *kc, *vc;
    const int32_t *row_slot, *row_pos;
    int T, H, G, dim, vdim, kp, vp, n_slots, max_len;
    float eps; int unit_rms;
};
template <typename E>
__global__ __launch_bounds__(256) void ob_sig_prep_kernel(const ObSigPrepArgs A)
{
    const int lane = threadIdx.x & 63;
    const int unit = blockIdx.x * 4 + (threadIdx.x >> 6), row = A.row0 + blockIdx.y;
    if (unit >= A.H + 2 * A.G) return;
    const int slot = A.row_slot[row], pos = A.row_pos[row];
    if (slot < 0 || slot >= A.n_slots || pos < 0 || pos >= A.max_len) return;
    const int kind = unit < A.H ? 0 : unit < A.H + A.G ? 1 : 2, h = kind == 0 ? unit : kind == 1 ? unit - A.H : unit - A.H - A.G;
    const int n = kind == 2 ? A.vdim : A.dim, np = kind == 2 ? A.vp : A.kp;
    const E *src = (const E *)A.u + (size_t)row * A.ldu + (kind == 0 ? h * A.dim : kind == 1 ? (A.H + h) * A.dim : (A.H + A.G) * A.dim + h * A.vdim);
    E *dst = kind == 0 ? (E *)A.qn + ((size_t)row * A.H + h) * A.kp
                       : (E *)(kind == 1 ? A.kc : A.vc) + (((size_t)slot * A.G + h) * A.max_len + pos) * np;
    float f = 1.f;
    if (kind < 2 && A.unit_rms) {
        float ss = 0.f;
        for (int d = lane; d < n; d += 64) { const float v = (float)src[d]; ss = __builtin_fmaf(v, v, ss); }
        f = 1.0f / sqrtf(ob_wave_sum(ss) / (float)n + A.eps);
    }
    for (int d = lane; d < np; d += 64) dst[d] = d < n ? (E)((float)src[d] * f) : (E)0.f;
}

// the same for bf16 heads of whole 16-byte pieces (dim % 8 == vdim % 8 == 0), padded to DP: DP / 8 lanes per head, one piece each
template <int DP>
__global__ __launch_bounds__(256) void ob_sig_prep_vec_kernel(const ObSigPrepArgs A)
{
    constexpr int LPH = DP / 8;
    const int i = blockIdx.x * 256 + threadIdx.x, unit = i / LPH, ds = i % LPH, row = A.row0 + blockIdx.y;
    const int slot = A.row_slot[row], pos = A.row_pos[row];
    if (slot < 0 || slot >= A.n_slots || pos < 0 || pos >= A.max_len) return;                          // (uniform)
    const bool live = unit < A.H + 2 * A.G;
    const int kind = unit < A.H ? 0 : unit < A.H + A.G ? 1 : 2, h = kind == 0 ? unit : kind == 1 ? unit - A.H : unit - A.H - A.G;
    const int n = kind == 2 ? A.vdim : A.dim;
    ob_bf8 v = (ob_bf8)(__bf16)0.f;
    if (live && 8 * ds < n)
        v = *reinterpret_cast<const ob_bf8 *>((const __bf16 *)A.u + (size_t)row * A.ldu +
                                              (kind < 2 ? unit * A.dim : (A.H + A.G) * A.dim + h * A.vdim) + 8 * ds);
    float ss = 0.f;
#pragma unroll
    for (int e = 0; e < 8; ++e) ss = __builtin_fmaf((float)v[e], (float)v[e], ss);
    ss += OB_DPP_F(ss, 0xB1, 0xF);
    ss += OB_DPP_F(ss, 0x4E, 0xF);
    ss += OB_DPP_F(ss, 0x141, 0xF);
    if (LPH == 16) ss += OB_DPP_F(ss, 0x140, 0xF);
    if (kind < 2 && A.unit_rms) {
        const float f = 1.0f / sqrtf(ss / (float)n + A.eps);
#pragma unroll
        for (int e = 0; e < 8; ++e) v[e] = (__bf16)((float)v[e] * f);
    }
    if (!live) return;
    __bf16 *dst = kind == 0 ? (__bf16 *)A.qn + ((size_t)row * A.H + h) * DP
                            : (__bf16 *)(kind == 1 ? A.kc : A.vc) + (((size_t)slot * A.G + h) * A.max_len + pos) * DP;
    *reinterpret_cast<ob_bf8 *>(dst + 8 * ds) = v;
}

// ---- any element type / head size: one workgroup per (row, head), fp32 arithmetic with the accurate functions
struct ObSigRowsArgs {
    const void *qn, *kc, *vc;
    void *out; int out_nkt;                    // fragment-major rows of the output product: column h vdim + d
    const int32_t *row_slot, *row_pos;
    int row0, H, G, dim, vdim, kp, vp, n_slots, max_len;
    float scale; ObSigBias b;
};
template <typename E>
__global__ __launch_bounds__(256) void ob_sig_rows_kernel(const ObSigRowsArgs A)
{
    __shared__ float ws[256];
    extern __shared__ float qs[];              // [dim]
    const int h = blockIdx.x, row = A.row0 + blockIdx.y, tid = threadIdx.x;
    const int slot = A.row_slot[row], pos = A.row_pos[row];
    if (slot < 0 || slot >= A.n_slots || pos < 0 || pos >= A.max_len) return;
    const int kvh = h / (A.H / A.G);
    const E *q = (const E *)A.qn + ((size_t)row * A.H + h) * A.kp;
    const E *kb = (const E *)A.kc + ((size_t)slot * A.G + kvh) * A.max_len * A.kp;
    const E *vb = (const E *)A.vc + ((size_t)slot * A.G + kvh) * A.max_len * A.vp;
    for (int d = tid; d < A.dim; d += 256) qs[d] = (float)q[d];
    const float r1 = A.b.r1 ? A.b.r1[h] : 0.f, r2 = A.b.r1 ? A.b.r2[h] : 0.f, pb = A.b.pb ? A.b.pb[h] : 0.f;
    E *out = (E *)A.out;
    for (int d0 = 0; d0 < A.vdim; d0 += 256) {                 // (one pass up to 256 value columns)
        const int d = d0 + tid;
        float o = 0.f;
        for (int j0 = 0; j0 <= pos; j0 += 256) {
            __syncthreads();
            const int j = j0 + tid;
            float w = 0.f;
            if (j <= pos) {
                const E *k = kb + (size_t)j * A.kp;
                float s = 0.f;
                for (int e = 0; e < A.dim; ++e) s = __builtin_fmaf((float)k[e], qs[e], s);
                w = ob_sigmoidf(s * A.scale - r1 * log1pf(r2 * (float)(pos - j)) + pb);
            }
            ws[tid] = w;
            __syncthreads();
            if (d < A.vdim) {
                const int nj = min(256, pos + 1 - j0);
                const E *v = vb + (size_t)j0 * A.vp + d;
                for (int jj = 0; jj < nj; ++jj) o = __builtin_fmaf(ws[jj], (float)v[(size_t)jj * A.vp], o);
            }
        }
        if (d < A.vdim) out[ob_frag<E>(row, h * A.vdim + d, A.out_nkt)] = (E)o;
    }
}

// ---- decode, bf16, padded head size DP = 64 / 128: R query heads of one kv head per workgroup, one key block ("split") of the context.
// DP / 8 lanes share a key (16 bytes each), the workgroup sweeps 2048 / DP keys at a time, NI sweeps in flight; q, k of the new token are
// brought to unit RMS here, the split that holds its position takes key and value from LDS and (one workgroup per kv head) appends them.
struct ObSigDecArgs {
    const void *u; int ldu, row0;
    void *kc, *vc;
    void *out; int out_nkt;
    const int32_t *row_slot, *row_pos;
    int H, G, dim, vdim, n_slots, max_len, chunk, nsplit;
    float scale, eps; ObSigBias b; int unit_rms;
    float *part; int *ticket;                  // [rows][H][nsplit][DP], [rows][head groups]; tickets zero between launches
};

template <int DP, int R>
__global__ __launch_bounds__(256) void ob_sig_dec_kernel(const ObSigDecArgs A)
{
    constexpr int LPK = DP / 8, PG = 256 / LPK, NI = 4;
    __shared__ __attribute__((aligned(16))) float po[4][R][DP];
    __shared__ __attribute__((aligned(16))) float q_s[R][DP];
    __shared__ __attribute__((aligned(16))) __bf16 kv_s[2][DP];
    __shared__ int last_s;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int row = A.row0 + blockIdx.y, split = blockIdx.z;
    const int slot = A.row_slot[row], pos = A.row_pos[row];
    if (slot < 0 || slot >= A.n_slots || pos < 0 || pos >= A.max_len) return;          // idle row (uniform)
    const int L = pos + 1, p_lo = split * A.chunk;
    if (p_lo >= L) return;                                                             // empty split (uniform)
    const int p_hi = min(L, p_lo + A.chunk), nlive = (L + A.chunk - 1) / A.chunk;
    const int rep = A.H / A.G, gpk = (rep + R - 1) / R;                                // workgroups per kv head
    const int kvh = blockIdx.x / gpk, h0 = kvh * rep + (blockIdx.x % gpk) * R, nh = min(R, (kvh + 1) * rep - h0);
    const int ds = tid & (LPK - 1), pg = tid / LPK;
    const size_t head_off = ((size_t)slot * A.G + kvh) * A.max_len * DP;
    const __bf16 *kb = (const __bf16 *)A.kc + head_off + 8 * ds, *vb = (const __bf16 *)A.vc + head_off + 8 * ds;
    ob_bf8 k8[NI], v8[NI], kn[NI], vn[NI];
    auto fetch = [&](ob_bf8 (&kd)[NI], ob_bf8 (&vd)[NI], int base) {
#pragma unroll
        for (int i = 0; i < NI; ++i) {
            const size_t off = (size_t)min(base + pg + PG * i, p_hi - 1) * DP;       // (never a row this request has not written)
            kd[i] = __builtin_nontemporal_load(reinterpret_cast<const ob_bf8 *>(kb + off));
            vd[i] = __builtin_nontemporal_load(reinterpret_cast<const ob_bf8 *>(vb + off));
        }
    };
    fetch(k8, v8, p_lo);                                                               // in flight while the query is formed
    const bool own_new = split == nlive - 1;                                           // (uniform) this split holds `pos`
    for (int role = wave; role < nh + (own_new ? 2 : 0); role += 4) {                  // R queries | key | value, one wave each
        const int kind = role < nh ? 0 : role - nh + 1, n = kind == 2 ? A.vdim : A.dim;
        const __bf16 *src = (const __bf16 *)A.u + (size_t)row * A.ldu +
                            (kind == 0 ? (h0 + role) * A.dim : kind == 1 ? (A.H + kvh) * A.dim : (A.H + A.G) * A.dim + kvh * A.vdim);
        float e[DP / 64], ss = 0.f;
#pragma unroll
        for (int c = 0; c < DP / 64; ++c) {
            const int d = lane + 64 * c;
            e[c] = d < n ? (float)src[d] : 0.f;
            ss = __builtin_fmaf(e[c], e[c], ss);
        }
        float f = 1.f;
        if (kind < 2 && A.unit_rms) f = 1.0f / sqrtf(ob_wave_sum(ss) / (float)n + A.eps);
#pragma unroll
        for (int c = 0; c < DP / 64; ++c) {
            const int d = lane + 64 * c;
            if (kind == 0) q_s[role][d] = e[c] * f * (-A.scale * OB_LOG2E);
            else {
                const __bf16 b = (__bf16)(e[c] * f);
                kv_s[kind - 1][d] = b;
                if (h0 == kvh * rep) ((__bf16 *)(kind == 1 ? A.kc : A.vc))[head_off + (size_t)pos * DP + d] = b;
            }
        }
    }
    __syncthreads();
    float q[R][8];
    float r1[R], r2[R], pb[R];
#pragma unroll
    for (int r = 0; r < R; ++r) {
        const int h = h0 + min(r, nh - 1);
#pragma unroll
        for (int e = 0; e < 8; ++e) q[r][e] = q_s[min(r, nh - 1)][8 * ds + e];
        r1[r] = A.b.r1 ? A.b.r1[h] : 0.f; r2[r] = A.b.r1 ? A.b.r2[h] : 0.f;
        pb[r] = A.b.pb ? A.b.pb[h] * OB_LOG2E : 0.f;
    }
    ob_bf8 kn8, vn8;
    if (own_new) {
        kn8 = *reinterpret_cast<const ob_bf8 *>(&kv_s[0][8 * ds]);
        vn8 = *reinterpret_cast<const ob_bf8 *>(&kv_s[1][8 * ds]);
    }
    float o[R][8];
#pragma unroll
    for (int r = 0; r < R; ++r)
#pragma unroll
        for (int e = 0; e < 8; ++e) o[r][e] = 0.f;
    for (int base = p_lo; base < p_hi; base += PG * NI) {
        const bool more = base + PG * NI < p_hi;                                       // (uniform)
        if (more) fetch(kn, vn, base + PG * NI);
#pragma unroll
        for (int i = 0; i < NI; ++i) {
            const int p = base + pg + PG * i;
            if (own_new && p >= pos) { k8[i] = kn8; v8[i] = vn8; }                     // (another workgroup writes the cache row `pos`)
            float kf[8], vf[8];
#pragma unroll
            for (int e = 0; e < 8; ++e) { kf[e] = (float)k8[i][e]; vf[e] = (float)v8[i][e]; }
            const float dist = (float)max(pos - p, 0);
#pragma unroll
            for (int r = 0; r < R; ++r) {
                float s = 0.f;
#pragma unroll
                for (int e = 0; e < 8; ++e) s = __builtin_fmaf(q[r][e], kf[e], s);
                s += OB_DPP_F(s, 0xB1, 0xF);                                           // over the key's LPK lanes
                s += OB_DPP_F(s, 0x4E, 0xF);
                s += OB_DPP_F(s, 0x141, 0xF);
                if (LPK == 16) s += OB_DPP_F(s, 0x140, 0xF);
                const float a = s + (r1[r] * __builtin_amdgcn_logf(__builtin_fmaf(r2[r], dist, 1.0f)) - pb[r]);
                const float w = p < p_hi ? __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(a)) : 0.f;
#pragma unroll
                for (int e = 0; e < 8; ++e) o[r][e] = __builtin_fmaf(w, vf[e], o[r][e]);
            }
        }
        if (more) {
#pragma unroll
            for (int i = 0; i < NI; ++i) { k8[i] = kn[i]; v8[i] = vn[i]; }
        }
    }
    // ---- the workgroup's key groups add up: lanes of a wave that share ds, then the four waves
#pragma unroll
    for (int r = 0; r < R; ++r) {
#pragma unroll
        for (int e = 0; e < 8; ++e) {
            float v = o[r][e];
#pragma unroll
            for (int s = LPK; s < 64; s <<= 1) v += __shfl_xor(v, s);
            if (lane < LPK) po[wave][r][8 * ds + e] = v;
        }
    }
    __syncthreads();
    __bf16 *out = (__bf16 *)A.out;
    if (nlive == 1) {                                                                  // (uniform)
        for (int i = tid; i < nh * DP; i += 256) {
            const int r = i / DP, d = i % DP;
            if (d < A.vdim) out[ob_frag<__bf16>(row, (h0 + r) * A.vdim + d, A.out_nkt)] = (__bf16)((po[0][r][d] + po[1][r][d]) + (po[2][r][d] + po[3][r][d]));
        }
        return;
    }
    // ---- publish this split's partial write-through, take a ticket; the last arriver adds them in split order
    float *pp = A.part + ((size_t)row * A.H + h0) * A.nsplit * DP;
    for (int i = tid; i < nh * DP; i += 256) {
        const int r = i / DP, d = i % DP;
        __hip_atomic_store(pp + ((size_t)r * A.nsplit + split) * DP + d, (po[0][r][d] + po[1][r][d]) + (po[2][r][d] + po[3][r][d]),
                           __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
    }
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");                                   // every wave: its stores have left
    __syncthreads();
    if (tid == 0) {
        int *tk = A.ticket + (size_t)row * gridDim.x + blockIdx.x;
        const int prev = __hip_atomic_fetch_add(tk, 1, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
        last_s = prev == nlive - 1;
        if (prev == nlive - 1) __hip_atomic_store(tk, 0, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
    }
    __syncthreads();
    if (!last_s) return;
    for (int i = tid; i < nh * DP; i += 256) {
        const int r = i / DP, d = i % DP;
        const float *ps = pp + (size_t)r * A.nsplit * DP + d;
        float acc = 0.f;
        for (int s0 = 0; s0 < nlive; s0 += 8) {
            float v[8];
#pragma unroll
            for (int j = 0; j < 8; ++j) v[j] = __hip_atomic_load(ps + (size_t)min(s0 + j, nlive - 1) * DP, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
#pragma unroll
            for (int j = 0; j < 8; ++j) if (s0 + j < nlive) acc += v[j];
        }
        if (d < A.vdim) out[ob_frag<__bf16>(row, (h0 + r) * A.vdim + d, A.out_nkt)] = (__bf16)acc;
    }
}
