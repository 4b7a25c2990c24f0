// State-space mixer (scalar decay per head and token; B / C shared by the heads of a group) with a causal convolution in front:
//   xbc_t = silu(bias + sum_j taps[:, j] in_{t - (n - 1) + j}),   dt = softplus(raw + dt_bias),   decay = exp(-exp(A_log) dt)
//   S_t = decay S_{t-1} + dt B_t x_t^T  (N x P, fp32),   y_t = S_t^T C_t + D x_t
// Everything but the projections and the convolution's activations is fp32; where prompt chunks run on MFMA the fp32 factors (state,
// decayed scores, weighted inputs) enter as two bf16 terms (hi + lo: 16 bits of mantissa) against the bf16 x / B / C.
//
// State per slot: S [heads][N][sp] fp32 (sp = P rounded up to 4, padding zero) and a ring of the convolution's inputs, token p at index
// p % taps ([taps][ch] elements): the newest token goes where no reader of this step looks, so every workgroup of a decode step may read
// its neighbours' channels while their owners append.  A request starts at position 0 with zeros: slots need no clearing.
//
//   ob_ssm_step_kernel   a run of tokens of one request per (head, 32-column slice), token by token: the decode step (one token, with the
//                        convolution fused) and fp32 prompts (after ob_conv_kernel)
//   ob_ssd_kernel        prompt rows in bf16, chunks of 64 tokens: inside a chunk the recurrence is two masked matrix products, between
//                        chunks the fp32 state is carried in accumulator registers
#pragma once
#include "ob_dense.h"

struct ObSsmArgs {
    const void *u; int ldu, x_off;             // input product rows; the convolution's input channels start at column x_off
    const void *xbc; int ldxbc;                // convolved rows (NULL: convolve here, single-token runs only)
    const float *aux; int ldaux;               // raw dt, fp32
    const float *conv_w, *conv_b;              // [taps][ch] (transposed), [ch]
    const float *dt_bias, *A_log, *D;          // [heads]
    float *state; void *ring;
    void *y; int ldy;
    const int32_t *row_slot, *row_pos;
    int row0;                                  // runs: row0 + blockIdx.y (single tokens) or the segment table
    int heads, groups, N, P, sp, taps, ch, n_slots, max_len;
};

#define OB_SSM_MAXSEG 64
struct ObSsmSeg { int row0, n, slot, past; };
struct ObSsmSegs { int nseg; ObSsmSeg s[OB_SSM_MAXSEG]; };

// The convolution's inputs of a finished run enter the ring: the last min(n, taps) tokens of channels [c0, c0 + nc)
template <typename E>
__device__ __forceinline__ void ob_ring_append(const ObSsmArgs &A, const ObSsmSeg &sg, int c0, int nc, int tid, int nthr)
{
    const int keep = min(sg.n, A.taps);
    for (int i = tid; i < keep * nc; i += nthr) {
        const int j = i / nc, c = c0 + i - j * nc, t = sg.n - keep + j;
        ((E *)A.ring)[((size_t)sg.slot * A.taps + (sg.past + t) % A.taps) * A.ch + c] = ((const E *)A.u)[(size_t)(sg.row0 + t) * A.ldu + A.x_off + c];
    }
}

// ---- the convolution of prompt rows: VEC channels per thread; row_off = tokens of the row's run before it
template <typename E, int VEC>
__global__ __launch_bounds__(256) void ob_conv_kernel(const ObSsmArgs A, const int32_t *__restrict__ row_off, void *xbc)
{
    const int row = A.row0 + blockIdx.y, c = (blockIdx.x * 256 + threadIdx.x) * VEC;
    const int slot = A.row_slot[row], pos = A.row_pos[row], off = row_off[row];
    if (c >= A.ch || slot < 0 || slot >= A.n_slots) return;
    float acc[VEC];
#pragma unroll
    for (int e = 0; e < VEC; ++e) acc[e] = A.conv_b[c + e];
    for (int b = 0; b < A.taps && b <= pos; ++b) {                 // b tokens back
        const E *src = b <= off ? (const E *)A.u + (size_t)(row - b) * A.ldu + A.x_off + c
                                : (const E *)A.ring + ((size_t)slot * A.taps + (pos - b) % A.taps) * A.ch + c;
        const float *w = A.conv_w + (size_t)(A.taps - 1 - b) * A.ch + c;
        E v[VEC];
        if constexpr (VEC * sizeof(E) == 16) *reinterpret_cast<typename ObElem<E>::V16 *>(v) = *reinterpret_cast<const typename ObElem<E>::V16 *>(src);
        else v[0] = src[0];
#pragma unroll
        for (int e = 0; e < VEC; ++e) acc[e] = __builtin_fmaf(w[e], (float)v[e], acc[e]);
    }
    E *o = (E *)xbc + (size_t)row * A.ldxbc + c;
    E r[VEC];
#pragma unroll
    for (int e = 0; e < VEC; ++e) r[e] = (E)ob_silu<E>(acc[e]);
    if constexpr (VEC * sizeof(E) == 16) *reinterpret_cast<typename ObElem<E>::V16 *>(o) = *reinterpret_cast<const typename ObElem<E>::V16 *>(r);
    else o[0] = r[0];
}

// the same for 2 to 4 taps: OB_CONV_ROWS rows per thread, the window of inputs sliding through registers (rebuilt where a run starts)
#define OB_CONV_ROWS 8
template <typename E, int TAPS>
__global__ __launch_bounds__(256) void ob_conv_rows_kernel(const ObSsmArgs A, const int32_t *__restrict__ row_off, void *xbc, int row_end)
{
    typedef typename ObElem<E>::V16 V16;
    constexpr int VEC = ObElem<E>::EPL, R = OB_CONV_ROWS;
    const int row0 = A.row0 + blockIdx.y * R, c = (blockIdx.x * 256 + threadIdx.x) * VEC;
    if (c >= A.ch) return;
    const E *u = (const E *)A.u + A.x_off + c;
    V16 in[R + TAPS - 1];                                          // in[TAPS - 1 + r] = row row0 + r
#pragma unroll
    for (int r = 0; r < R; ++r) in[TAPS - 1 + r] = *reinterpret_cast<const V16 *>(u + (size_t)min(row0 + r, row_end - 1) * A.ldu);
    float w[TAPS][VEC], b[VEC];
#pragma unroll
    for (int e = 0; e < VEC; ++e) b[e] = A.conv_b[c + e];
#pragma unroll
    for (int t = 0; t < TAPS; ++t)
#pragma unroll
        for (int e = 0; e < VEC; ++e) w[t][e] = A.conv_w[(size_t)t * A.ch + c + e];
#pragma unroll
    for (int r = 0; r < R; ++r) {
        const int row = row0 + r;
        if (row >= row_end) break;
        const int off = row_off[row];
        V16 x[TAPS];                                               // x[t]: TAPS - 1 - t tokens back
#pragma unroll
        for (int t = 0; t < TAPS; ++t) x[t] = in[r + t];
        if (off < TAPS - 1 || r < TAPS - 1) {                      // (uniform) some of the window lies before the run or the thread's rows
            const int slot = A.row_slot[row], pos = A.row_pos[row];
#pragma unroll
            for (int t = 0; t < TAPS - 1; ++t) {
                const int back = TAPS - 1 - t;
                if (back > pos) x[t] = (V16)(E)0.f;
                else if (back > off) x[t] = *reinterpret_cast<const V16 *>((const E *)A.ring + ((size_t)slot * A.taps + (pos - back) % A.taps) * A.ch + c);
                else if (r < back) x[t] = *reinterpret_cast<const V16 *>(u + (size_t)(row - back) * A.ldu);
            }
        }
        V16 o;
#pragma unroll
        for (int e = 0; e < VEC; ++e) {
            float acc = b[e];
#pragma unroll
            for (int t = TAPS - 1; t >= 0; --t) acc = __builtin_fmaf(w[t][e], (float)x[t][e], acc);
            o[e] = (E)ob_silu<E>(acc);
        }
        *reinterpret_cast<V16 *>((E *)xbc + (size_t)row * A.ldxbc + c) = o;
    }
}

// ---- token by token.  Thread = (4 state columns, every 32nd state row): NI rows in registers
template <typename E, int NI>
__global__ __launch_bounds__(256) void ob_ssm_step_kernel(const ObSsmArgs A, const ObSsmSegs SG)
{
    constexpr int NMAX = NI * 32;
    __shared__ __attribute__((aligned(16))) float xs[32], Bs[NMAX], Cs[NMAX];
    __shared__ __attribute__((aligned(16))) ob_float4 ys[32][8];
    const int tid = threadIdx.x, pc = tid & 7, ng = tid >> 3;
    const int nsl = (A.P + 31) >> 5, h = blockIdx.x / nsl, p0 = (blockIdx.x % nsl) * 32;
    ObSsmSeg sg;
    if (SG.nseg > 0) sg = SG.s[blockIdx.y];
    else { const int r = A.row0 + blockIdx.y; sg = {r, 1, A.row_slot[r], A.row_pos[r]}; }
    if (sg.slot < 0 || sg.slot >= A.n_slots || sg.past < 0 || sg.past >= A.max_len) return;        // idle row (uniform)
    const int g = h / (A.heads / A.groups), inner = A.heads * A.P, GN = A.groups * A.N;
    const int p = p0 + 4 * pc;
    const bool pok = p < A.sp;
    float *st = A.state + (((size_t)sg.slot * A.heads + h) * A.N) * A.sp + p;
    ob_float4 S[NI];
#pragma unroll
    for (int i = 0; i < NI; ++i) {
        const int n = ng + 32 * i;
        S[i] = (ob_float4){0.f, 0.f, 0.f, 0.f};
        if (sg.past > 0 && pok && n < A.N) S[i] = __builtin_nontemporal_load(reinterpret_cast<const ob_float4 *>(st + (size_t)n * A.sp));
    }
    const float dtb = A.dt_bias[h], na = -expf(A.A_log[h]), Dh = A.D[h];
    const int npx = min(32, A.P - p0), nch = npx + 2 * A.N;
    auto chan = [&](int i) { return i < npx ? h * A.P + p0 + i : i < npx + A.N ? inner + g * A.N + (i - npx) : inner + GN + g * A.N + (i - npx - A.N); };
    for (int t = 0; t < sg.n; ++t) {
        const int row = sg.row0 + t, pos = sg.past + t;
        if (t == 0 && npx < 32) for (int i = tid; i < 32; i += 256) xs[i] = 0.f;
        if (t > 0 || npx < 32) __syncthreads();
        for (int i = tid; i < nch; i += 256) {
            const int c = chan(i);
            float v;
            if (A.xbc) v = (float)((const E *)A.xbc)[(size_t)row * A.ldxbc + c];
            else {
                const E cur = ((const E *)A.u)[(size_t)row * A.ldu + A.x_off + c];
                E *rg = (E *)A.ring + (size_t)sg.slot * A.taps * A.ch + c;
                float acc = A.conv_b[c];
                for (int b = 0; b < A.taps && b <= pos; ++b)
                    acc = __builtin_fmaf(A.conv_w[(size_t)(A.taps - 1 - b) * A.ch + c], b ? (float)rg[(size_t)((pos - b) % A.taps) * A.ch] : (float)cur, acc);
                if (i < npx || (p0 == 0 && h % (A.heads / A.groups) == 0)) rg[(size_t)(pos % A.taps) * A.ch] = cur;
                v = (float)(E)ob_silu<E>(acc);
            }
            (i < npx ? xs[i] : i < npx + A.N ? Bs[i - npx] : Cs[i - npx - A.N]) = v;
        }
        __syncthreads();
        const float dt = ob_softplusf(A.aux[(size_t)row * A.ldaux + h] + dtb), dec = expf(na * dt);
        const ob_float4 x4 = *reinterpret_cast<const ob_float4 *>(&xs[4 * pc]);
        ob_float4 y = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int i = 0; i < NI; ++i) {
            const int n = ng + 32 * i;
            if (n < A.N) {
                const float db = dt * Bs[n], c = Cs[n];
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    S[i][e] = __builtin_fmaf(db, x4[e], dec * S[i][e]);
                    y[e] = __builtin_fmaf(c, S[i][e], y[e]);
                }
            }
        }
        ys[ng][pc] = y;
        __syncthreads();
        if (tid < npx) {
            const float *yc = reinterpret_cast<const float *>(ys) + tid;           // column tid of the 32 partial rows
            float s[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int k = 0; k < 32; ++k) s[k & 3] += yc[32 * k];
            ((E *)A.y)[(size_t)row * A.ldy + h * A.P + p0 + tid] = (E)__builtin_fmaf(Dh, xs[tid], (s[0] + s[1]) + (s[2] + s[3]));
        }
    }
#pragma unroll
    for (int i = 0; i < NI; ++i) {
        const int n = ng + 32 * i;
        if (pok && n < A.N) __builtin_nontemporal_store(S[i], reinterpret_cast<ob_float4 *>(st + (size_t)n * A.sp));
    }
    if (A.xbc) {
        ob_ring_append<E>(A, sg, h * A.P + p0, npx, tid, 256);
        if (p0 == 0 && h % (A.heads / A.groups) == 0) {
            ob_ring_append<E>(A, sg, inner + g * A.N, A.N, tid, 256);
            ob_ring_append<E>(A, sg, inner + GN + g * A.N, A.N, tid, 256);
        }
    }
}

// ---- chunks of 64 tokens on MFMA (bf16 x / B / C).  Workgroup = (segment, head, 32 state columns), 4 waves; NP = N padded.
//   G^T[s][t] = B_s . C_t (wave w: tokens 16 w ..), masked and decayed in registers -> it IS the B operand of Y^T += X^T M^T
//   Y^T[p][t] = (S_prev^T C_t) exp(cum_t) + X^T M^T + D x;   S <- exp(cum_63) S + B^T (x dt exp(cum_63 - cum))
// The kernel is bound by VALU issue (two waves per SIMD): decays live in the base-2 domain, the weighted inputs x dt exp(..) are formed once
// per element on their way into LDS, splits into bf16 terms cost three operations per element, tiles above the diagonal none.
// LDS rows of 128 / 256 columns are unpadded, 16-byte pieces XOR-swizzled by the row: piece pc of row r sits at pc ^ f(r), f(r) = 2 m + (r >> 3),
// m = r for rows 0 .. 7 and (r - 8) ^ 4 for rows 8 .. 15.  Operand reads (a ds_read_b128 lane group = rows {0-3, 12-15} at one piece and rows
// 4-11 at the next) and transpose reads (a half-wave = two adjacent pieces of 8 rows) then both cover the 64 banks once.
template <int NP> __device__ __forceinline__ int ob_ssd_at(int r, int k)      // element offset of (row, column) in such a tile
{
    if constexpr (NP < 128) return r * (NP + 8) + k;                          // (64 columns: padded rows)
    else {
        const int r16 = r & 15, f = 2 * (r16 < 8 ? r16 : (r16 & 7) ^ 4) + (r16 >> 3);
        return r * NP + ((((k >> 3) ^ f) << 3) | (k & 7));
    }
}
template <int NP, bool VEC>
__global__ __launch_bounds__(256) void ob_ssd_kernel(const ObSsmArgs A, const ObSsmSegs SG)
{
    typedef short ob_v4s __attribute__((ext_vector_type(4)));
    typedef short ob_v8s __attribute__((ext_vector_type(8)));
    typedef __attribute__((address_space(3))) ob_v4s ob_lds_v4s;
    constexpr int Q = 64, LD = NP < 128 ? NP + 8 : NP, LX = 48, KN = NP / 32, NT = NP / 32;     // n tiles per wave: NP / 16 / 2
    __shared__ __attribute__((aligned(16))) __bf16 Bs[Q * LD], Cs[Q * LD], Xs[Q][LX], Xh[Q][LX], Xl[Q][LX], Sh[32 * LD], Sl[32 * LD];
    __shared__ __attribute__((aligned(16))) float cum2[2][Q], dts2[2][Q], wgt2[2][Q];
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), lr = lane & 15, g4 = lane >> 4;
    const int nsl = (A.P + 31) >> 5, h = blockIdx.x / nsl, p0 = (blockIdx.x % nsl) * 32, npx = min(32, A.P - p0);
    const ObSsmSeg sg = SG.s[blockIdx.y];
    const int grp = h / (A.heads / A.groups), inner = A.heads * A.P, GN = A.groups * A.N;
    const __bf16 *xb = (const __bf16 *)A.xbc + (size_t)sg.row0 * A.ldxbc;
    const int cx = h * A.P + p0, cB = inner + grp * A.N, cC = inner + GN + grp * A.N;
    const float dtb = A.dt_bias[h], na = -1.4426950408889634f * expf(A.A_log[h]), Dh = A.D[h];
    float *st = A.state + (((size_t)sg.slot * A.heads + h) * A.N) * A.sp;
    // state: wave = (p tile wave & 1, n tiles (wave >> 1) NT ..); lane holds column p = lr, rows n = 4 g4 .. + 3
    const int pt = wave & 1, nt0 = (wave >> 1) * NT, pcol = p0 + 16 * pt + lr;
    ob_float4 S[NT];
#pragma unroll
    for (int i = 0; i < NT; ++i)
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const int n = 16 * (nt0 + i) + 4 * g4 + e;
            S[i][e] = sg.past > 0 && n < A.N && pcol < A.P ? st[(size_t)n * A.sp + pcol] : 0.f;
        }
    // staging: pieces of 8 channels; rows past the run and channels past N / P are zero.  Thread: piece kp of rows tb + RB i of B and of C
    constexpr int NPC = NP / 8, PB = Q * NPC / 256, RB = 256 / NPC;
    const int tb = tid / NPC, kb = (tid % NPC) * 8, tx = tid >> 2, kx = (tid & 3) * 8;
    ob_u32x4 rb[PB], rc[PB], rx;
    float rdt = 0.f;
    auto piece = [&](const __bf16 *s, bool in, int k, int n) {           // 8 channels from s, of which n - k exist
        ob_u32x4 v = {0u, 0u, 0u, 0u};
        if (in && k < n) {
            if constexpr (VEC) v = *reinterpret_cast<const ob_u32x4 *>(s);
            else {
                ob_bf8 w = (ob_bf8)(__bf16)0.f;
#pragma unroll
                for (int e = 0; e < 8; ++e) if (k + e < n) w[e] = s[e];
                v = __builtin_bit_cast(ob_u32x4, w);
            }
        }
        return v;
    };
    const __bf16 *sB = xb + (size_t)tb * A.ldxbc + cB + kb, *sC = sB + (cC - cB), *sX = xb + (size_t)tx * A.ldxbc + cx + kx;
    const float *sD = A.aux + (size_t)(sg.row0 + lane) * A.ldaux + h;
    auto fetch = [&](int t0) {                                            // (called once per chunk, in order: the pointers advance)
#pragma unroll
        for (int i = 0; i < PB; ++i) {
            const bool in = t0 + tb + RB * i < sg.n;
            rb[i] = piece(sB + (size_t)(RB * i) * A.ldxbc, in, kb, A.N);
            rc[i] = piece(sC + (size_t)(RB * i) * A.ldxbc, in, kb, A.N);
        }
        rx = piece(sX, t0 + tx < sg.n, kx, npx);
        if (wave == 0) rdt = t0 + lane < sg.n ? *sD : 0.f;
        sB += (size_t)Q * A.ldxbc; sC += (size_t)Q * A.ldxbc; sX += (size_t)Q * A.ldxbc; sD += (size_t)Q * A.ldaux;
    };
    // a chunk's step sizes, summed log2 decays and input weights: wave 0 (whose tokens have the fewest predecessors) forms the NEXT chunk's
    // while the others still multiply
    auto decays = [&](int t0, int buf) {
        const float dt = t0 + lane < sg.n ? ob_softplusf(rdt + dtb) : 0.f;          // (no token: no decay, no input)
        float c = na * dt;
#pragma unroll
        for (int s = 1; s < 64; s <<= 1) { const float o = __shfl_up(c, s); if (lane >= s) c += o; }
        const float tot = __shfl(c, 63);
        cum2[buf][lane] = c; dts2[buf][lane] = dt; wgt2[buf][lane] = dt * __builtin_amdgcn_exp2f(tot - c);
    };
    fetch(0);
    if (wave == 0) decays(0, 0);
    __syncthreads();
    auto tr8 = [&](const __bf16 *lo_p, const __bf16 *hi_p) {             // two transpose reads: 4 + 4 rows of this lane's column
        const ob_v4s lo = __builtin_amdgcn_ds_read_tr16_b64_v4i16((ob_lds_v4s *)lo_p);
        const ob_v4s hi = __builtin_amdgcn_ds_read_tr16_b64_v4i16((ob_lds_v4s *)hi_p);
        return __builtin_bit_cast(ob_bf8, (ob_v8s){lo[0], lo[1], lo[2], lo[3], hi[0], hi[1], hi[2], hi[3]});
    };
    const int trow = 4 * g4 + (lr >> 2), tcol = 4 * (lr & 3);
    for (int t0 = 0; t0 < sg.n; t0 += Q) {
        const float *cum = cum2[(t0 / Q) & 1], *dts = dts2[(t0 / Q) & 1], *wgt = wgt2[(t0 / Q) & 1];
        // ---- this chunk's rows, its weighted inputs and the state's two terms into LDS
#pragma unroll
        for (int i = 0; i < PB; ++i) {
            *reinterpret_cast<ob_u32x4 *>(&Bs[ob_ssd_at<NP>(tb + RB * i, kb)]) = rb[i];
            *reinterpret_cast<ob_u32x4 *>(&Cs[ob_ssd_at<NP>(tb + RB * i, kb)]) = rc[i];
        }
        *reinterpret_cast<ob_u32x4 *>(&Xs[tx][kx]) = rx;
        {
            const float w = wgt[tx];
            ob_u32x4 xh, xl;
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                uint32_t hi, lo;
                ob_split_bf2(__uint_as_float(rx[e] << 16) * w, __uint_as_float(rx[e] & 0xffff0000u) * w, hi, lo);
                xh[e] = hi; xl[e] = lo;
            }
            *reinterpret_cast<ob_u32x4 *>(&Xh[tx][kx]) = xh;
            *reinterpret_cast<ob_u32x4 *>(&Xl[tx][kx]) = xl;
        }
#pragma unroll
        for (int i = 0; i < NT; ++i) {
            uint32_t h0, l0, h1, l1;
            ob_split_bf2(S[i][0], S[i][1], h0, l0);
            ob_split_bf2(S[i][2], S[i][3], h1, l1);
            *reinterpret_cast<ob_u32x2 *>(&Sh[ob_ssd_at<NP>(16 * pt + lr, 16 * (nt0 + i) + 4 * g4)]) = (ob_u32x2){h0, h1};
            *reinterpret_cast<ob_u32x2 *>(&Sl[ob_ssd_at<NP>(16 * pt + lr, 16 * (nt0 + i) + 4 * g4)]) = (ob_u32x2){l0, l1};
        }
        __syncthreads();
        if (t0 + Q < sg.n) fetch(t0 + Q);
        // ---- scores of this wave's 16 tokens against the tokens up to them
        ob_bf8 cf[KN];
#pragma unroll
        for (int k = 0; k < KN; ++k) cf[k] = *reinterpret_cast<const ob_bf8 *>(&Cs[ob_ssd_at<NP>(16 * wave + lr, 32 * k + 8 * g4)]);
        const int tq = 16 * wave + lr;
        const float ct = cum[tq];
        ob_u32x4 mh[2], ml[2];
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            uint32_t h0 = 0, l0 = 0, h1 = 0, l1 = 0;
            if (j <= wave) {                                     // (wave-uniform)
                ob_float4 a = {0.f, 0.f, 0.f, 0.f}, a1 = {0.f, 0.f, 0.f, 0.f};          // (two chains: a dependent MFMA waits for its predecessor)
#pragma unroll
                for (int k = 0; k < KN; k += 2) {
                    a = ObElem<__bf16>::mma(*reinterpret_cast<const ob_bf8 *>(&Bs[ob_ssd_at<NP>(16 * j + lr, 32 * k + 8 * g4)]), cf[k], a);
                    a1 = ObElem<__bf16>::mma(*reinterpret_cast<const ob_bf8 *>(&Bs[ob_ssd_at<NP>(16 * j + lr, 32 * k + 32 + 8 * g4)]), cf[k + 1], a1);
                }
                a += a1;
                const ob_float4 cs = *reinterpret_cast<const ob_float4 *>(&cum[16 * j + 4 * g4]), ds = *reinterpret_cast<const ob_float4 *>(&dts[16 * j + 4 * g4]);
                float m[4];
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    m[e] = a[e] * (ds[e] * __builtin_amdgcn_exp2f(ct - cs[e]));
                    if (j == wave && 4 * g4 + e > lr) m[e] = 0.f;
                }
                ob_split_bf2(m[0], m[1], h0, l0);
                ob_split_bf2(m[2], m[3], h1, l1);
            }
            mh[j >> 1][2 * (j & 1)] = h0; mh[j >> 1][2 * (j & 1) + 1] = h1;
            ml[j >> 1][2 * (j & 1)] = l0; ml[j >> 1][2 * (j & 1) + 1] = l1;
        }
        // ---- outputs
        const float ec = __builtin_amdgcn_exp2f(ct);
        ob_float4 ya[2][2];                                      // [p tile][hi, lo]: four independent chains
#pragma unroll
        for (int q = 0; q < 2; ++q) ya[q][0] = ya[q][1] = (ob_float4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int k = 0; k < KN; ++k)
#pragma unroll
            for (int q = 0; q < 2; ++q) {
                ya[q][0] = ObElem<__bf16>::mma(*reinterpret_cast<const ob_bf8 *>(&Sh[ob_ssd_at<NP>(16 * q + lr, 32 * k + 8 * g4)]), cf[k], ya[q][0]);
                ya[q][1] = ObElem<__bf16>::mma(*reinterpret_cast<const ob_bf8 *>(&Sl[ob_ssd_at<NP>(16 * q + lr, 32 * k + 8 * g4)]), cf[k], ya[q][1]);
            }
#pragma unroll
        for (int q = 0; q < 2; ++q) { ya[q][0] *= ec; ya[q][1] *= ec; }
#pragma unroll
        for (int s = 0; s < 2; ++s) {
            if (2 * s > wave) continue;
#pragma unroll
            for (int q = 0; q < 2; ++q) {
                const ob_bf8 xt = tr8(&Xs[32 * s + trow][16 * q + tcol], &Xs[32 * s + 16 + trow][16 * q + tcol]);
                ya[q][0] = ObElem<__bf16>::mma(xt, __builtin_bit_cast(ob_bf8, mh[s]), ya[q][0]);
                ya[q][1] = ObElem<__bf16>::mma(xt, __builtin_bit_cast(ob_bf8, ml[s]), ya[q][1]);
            }
        }
#pragma unroll
        for (int q = 0; q < 2; ++q) {
            ob_float4 y = ya[q][0] + ya[q][1];
            const ob_u32x2 xv = *reinterpret_cast<const ob_u32x2 *>(&Xs[tq][16 * q + 4 * g4]);
            const int p = 16 * q + 4 * g4;
            if (t0 + tq < sg.n) {
                __bf16 *o = (__bf16 *)A.y + (size_t)(sg.row0 + t0 + tq) * A.ldy + cx + p;
#pragma unroll
                for (int e = 0; e < 4; ++e) y[e] = __builtin_fmaf(Dh, __uint_as_float((e & 1) ? xv[e >> 1] & 0xffff0000u : xv[e >> 1] << 16), y[e]);
                if constexpr (VEC) { if (p < npx) *reinterpret_cast<ob_u32x2 *>(o) = (ob_u32x2){ob_pack_bf2(y[0], y[1]), ob_pack_bf2(y[2], y[3])}; }
                else { for (int e = 0; e < 4; ++e) if (p + e < npx) o[e] = (__bf16)y[e]; }
            }
        }
        // ---- the state behind the chunk
        const float et = __builtin_amdgcn_exp2f(cum[63]);
#pragma unroll
        for (int i = 0; i < NT; ++i) S[i] *= et;
#pragma unroll
        for (int s = 0; s < 2; ++s) {
            const ob_bf8 xh = tr8(&Xh[32 * s + trow][16 * pt + tcol], &Xh[32 * s + 16 + trow][16 * pt + tcol]);
            const ob_bf8 xl = tr8(&Xl[32 * s + trow][16 * pt + tcol], &Xl[32 * s + 16 + trow][16 * pt + tcol]);
#pragma unroll
            for (int i = 0; i < NT; ++i) {
                const ob_bf8 bt = tr8(&Bs[ob_ssd_at<NP>(32 * s + trow, 16 * (nt0 + i) + tcol)], &Bs[ob_ssd_at<NP>(32 * s + 16 + trow, 16 * (nt0 + i) + tcol)]);
                S[i] = ObElem<__bf16>::mma(bt, xh, S[i]);
                S[i] = ObElem<__bf16>::mma(bt, xl, S[i]);
            }
        }
        if (wave == 0 && t0 + Q < sg.n) decays(t0 + Q, ((t0 / Q) & 1) ^ 1);
        __syncthreads();                                         // every read of this chunk's LDS is complete
    }
#pragma unroll
    for (int i = 0; i < NT; ++i)
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const int n = 16 * (nt0 + i) + 4 * g4 + e;
            if (n < A.N && pcol < A.P) st[(size_t)n * A.sp + pcol] = S[i][e];
        }
    ob_ring_append<__bf16>(A, sg, cx, npx, tid, 256);
    if (p0 == 0 && h % (A.heads / A.groups) == 0) {
        ob_ring_append<__bf16>(A, sg, cB, A.N, tid, 256);
        ob_ring_append<__bf16>(A, sg, cC, A.N, tid, 256);
    }
}
