// Routing of a mixture of experts: which experts a token uses and with which weights, and the experts' row lists for the grouped products
// (ob_dense.h, OB_ROWS_GATHER / OB_ROWS_SORTED).
//   s = softmax(z) over experts and identity experts;  choice = s + correction;  of `groups` equal groups of neighbours only the `keep` with
//   the largest member count;  the `top` largest choices are used with weight s (not renormalised).  Identity experts (the last ones) return
//   their input: their weights add up to one factor per token.  Ties go to the smaller index.
// Results: tok_row / tok_w [T][top] = row of the sorted space (-1: none) and weight; id_w [T]; gather[row] = token; blk = row blocks of at most
// block_rows rows, an expert's first one at a multiple of 16 (empty blocks behind the last one, up to n_blk).
#pragma once
#include "ob_dense.h"

#define OB_MOE_TOKENS 64              // tokens per workgroup
struct ObRouteArgs {
    const float *z; int ldz;                   // router logits [T][experts + identity]
    const float *correction;
    int T, experts, identity, top, groups, keep;
    int32_t *tok_row; float *tok_w, *id_w;     // (tok_row holds the expert between the two passes)
    int32_t *hist;                             // [workgroups][experts]
    int32_t *gather; ObRowBlock *blk; int block_rows, n_blk;
};
// LDS of the first pass: per wave [groups] group maxima; [experts] counts; [64 top] experts of the workgroup's tokens
static inline size_t ob_route_lds(const ObRouteArgs &A) { return (16 * (size_t)A.groups + A.experts + (size_t)OB_MOE_TOKENS * A.top) * 4; }
#define OB_MOE_MAX 1024               // experts + identity experts

// order-preserving integers: the largest of a group through an LDS atomic
__device__ __forceinline__ uint32_t ob_ordered(float v) { const uint32_t u = __float_as_uint(v); return u & 0x80000000u ? ~u : u | 0x80000000u; }

// one wave per token, entry i = lane + 64 j in registers; z: its logits (-inf beyond N)
template <int NJ>
__device__ __forceinline__ void ob_route_token(const ObRouteArgs &A, int t, const float (&z)[NJ], const float (&corr)[NJ], uint32_t *gs, int *slots, int lane)
{
    const int N = A.experts + A.identity;
    float mx = z[0];
#pragma unroll
    for (int j = 1; j < NJ; ++j) mx = fmaxf(mx, z[j]);
    mx = ob_wave_max(mx);
    float p[NJ], c[NJ], sum = 0.f;
#pragma unroll
    for (int j = 0; j < NJ; ++j) { p[j] = expf(z[j] - mx); sum += p[j]; }
    const float inv = 1.0f / ob_wave_sum(sum);
#pragma unroll
    for (int j = 0; j < NJ; ++j) { p[j] *= inv; c[j] = lane + 64 * j < N ? p[j] + corr[j] : -INFINITY; }
    if (A.keep < A.groups) {
        const float per_inv = (float)A.groups / (float)N;
        auto fence = [] { __builtin_amdgcn_wave_barrier(); asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory"); };
        auto group = [&](int j) { return (int)(((float)(lane + 64 * j) + 0.5f) * per_inv); };         // (lane + 64 j) / (N / groups)
        for (int g = lane; g < A.groups; g += 64) gs[g] = 0;
        fence();
#pragma unroll
        for (int j = 0; j < NJ; ++j) if (lane + 64 * j < N) atomicMax(&gs[group(j)], ob_ordered(c[j]));
        fence();
#pragma unroll
        for (int j = 0; j < NJ; ++j) {
            if (lane + 64 * j >= N) continue;
            const int g = group(j);
            const uint32_t mine = gs[g];
            int r = 0;
            for (int o = 0; o < A.groups; ++o) r += gs[o] > mine || (gs[o] == mine && o < g);
            if (r >= A.keep) c[j] = -INFINITY;
        }
    }
    float idw = 0.f;
    for (int k = 0; k < A.top; ++k) {
        float best = c[0];
#pragma unroll
        for (int j = 1; j < NJ; ++j) best = fmaxf(best, c[j]);
        best = ob_wave_max(best);
        int at = -1;                                                  // the smallest index among equals (uniform); none left: -1
        float w = 0.f;
        if (best > -INFINITY) {
#pragma unroll
            for (int j = 0; j < NJ; ++j) {
                const uint64_t b = at < 0 ? __builtin_amdgcn_ballot_w64(c[j] == best) : 0;
                if (b) {
                    const int l = __builtin_ctzll(b);
                    at = l + 64 * j;
                    w = __builtin_bit_cast(float, __builtin_amdgcn_readlane(__builtin_bit_cast(int, p[j]), l));
                    if (lane == l) c[j] = -INFINITY;
                }
            }
        }
        if (at >= A.experts) { idw += w; at = -1; }
        if (lane == 0) { slots[k] = at; A.tok_w[(size_t)t * A.top + k] = w; }
    }
    if (lane == 0) A.id_w[t] = idw;
}

// offsets of the experts' rows and the block table from counts in LDS; 1024 threads.  cnt[e] -> first row of e.
__device__ __forceinline__ void ob_route_offsets(const ObRouteArgs &A, int *cnt, int *scan, int tid)
{
    // scan[2 w], scan[2 w + 1]: rows / blocks of the waves before; experts in runs of 1024
    int row_base = 0, blk_base = 0;
    for (int e0 = 0; e0 < A.experts; e0 += 1024) {
        const int e = e0 + tid, c = e < A.experts ? cnt[e] : 0;
        const int rows = (c + 15) & ~15, nb = (c + A.block_rows - 1) / A.block_rows;
        int r = rows, b = nb;
#pragma unroll
        for (int s = 1; s < 64; s <<= 1) {
            const int pr = __shfl_up(r, s), pb = __shfl_up(b, s);
            if ((tid & 63) >= s) { r += pr; b += pb; }
        }
        __syncthreads();
        if ((tid & 63) == 63) { scan[2 * (tid >> 6)] = r; scan[2 * (tid >> 6) + 1] = b; }
        __syncthreads();
        int r0 = row_base, b0 = blk_base;
        for (int w = 0; w < 16; ++w) {
            if (w < (tid >> 6)) { r0 += scan[2 * w]; b0 += scan[2 * w + 1]; }
            row_base += scan[2 * w]; blk_base += scan[2 * w + 1];
        }
        r0 += r - rows; b0 += b - nb;
        if (e < A.experts) {
            cnt[e] = r0;
            for (int k = 0; k < nb && b0 + k < A.n_blk; ++k) A.blk[b0 + k] = {e, r0 + k * A.block_rows, min(A.block_rows, c - k * A.block_rows), 0};
        }
    }
    for (int k = blk_base + tid; k < A.n_blk; k += 1024) A.blk[k] = {0, 0, 0, 0};
}

// first pass: choices, weights, and this workgroup's tokens per expert.  SINGLE: up to 64 tokens in one workgroup, everything in one launch.
template <bool SINGLE, int NJ>
__global__ __launch_bounds__(1024) void ob_route_kernel(const ObRouteArgs A)
{
    extern __shared__ __attribute__((aligned(16))) float sm[];
    __shared__ int scan[32];
    constexpr int PER = NJ <= 4 ? OB_MOE_TOKENS / 16 : 1;             // a wave's tokens whose logits are requested together
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), N = A.experts + A.identity;
    uint32_t *gs = reinterpret_cast<uint32_t *>(sm) + wave * A.groups;
    int *cnt = reinterpret_cast<int *>(sm) + 16 * A.groups, *slots = cnt + A.experts;
    for (int e = tid; e < A.experts; e += 1024) cnt[e] = 0;
    const int t0 = blockIdx.x * OB_MOE_TOKENS, t1 = min(A.T, t0 + OB_MOE_TOKENS), n = (t1 - t0) * A.top;
    float corr[NJ];
#pragma unroll
    for (int j = 0; j < NJ; ++j) corr[j] = lane + 64 * j < N ? A.correction[lane + 64 * j] : 0.f;
    for (int tb = t0 + wave; tb < t1; tb += 16 * PER) {
        float z[PER][NJ];
#pragma unroll
        for (int q = 0; q < PER; ++q)
#pragma unroll
            for (int j = 0; j < NJ; ++j)
                z[q][j] = tb + 16 * q < t1 && lane + 64 * j < N ? A.z[(size_t)(tb + 16 * q) * A.ldz + lane + 64 * j] : -INFINITY;
#pragma unroll 1
        for (int q = 0; q < PER; ++q) {
            const int t = tb + 16 * q;
            if (t >= t1) break;
            ob_route_token<NJ>(A, t, z[0], corr, gs, slots + (t - t0) * A.top, lane);
#pragma unroll
            for (int s = 0; s + 1 < PER; ++s)                         // (the next token's logits move up: one copy of the code)
#pragma unroll
                for (int j = 0; j < NJ; ++j) z[s][j] = z[s + 1][j];
        }
    }
    __syncthreads();
    for (int i = tid; i < n; i += 1024) if (slots[i] >= 0) atomicAdd(&cnt[slots[i]], 1);
    __syncthreads();
    if constexpr (!SINGLE) {
        for (int e = tid; e < A.experts; e += 1024) A.hist[(size_t)blockIdx.x * A.experts + e] = cnt[e];
        for (int i = tid; i < n; i += 1024) A.tok_row[(size_t)t0 * A.top + i] = slots[i];
    } else {
        ob_route_offsets(A, cnt, scan, tid);
        __syncthreads();
        for (int i = tid; i < n; i += 1024) {
            int r = -1;
            if (slots[i] >= 0) {
                r = atomicAdd(&cnt[slots[i]], 1);                     // (the order within an expert is free: every row is computed alone)
                A.gather[r] = i / A.top;
            }
            A.tok_row[i] = r;
        }
    }
}

// second pass, one workgroup: counts of all workgroups -> where each workgroup's tokens of an expert start; row and block tables.  An expert's
// workgroups are shared by `runs` threads (runs * experts <= 1024, or one run).
__global__ __launch_bounds__(1024) void ob_route_scan_kernel(const ObRouteArgs A, int n_wg, int runs)
{
    extern __shared__ int icnt[];                                     // [experts] | [runs][experts]
    __shared__ int scan[32];
    int *part = icnt + A.experts;
    const int tid = threadIdx.x, per = (n_wg + runs - 1) / runs;
    for (int i = tid; i < runs * A.experts; i += 1024) {
        const int q = i / A.experts, e = i - q * A.experts, b1 = min(n_wg, (q + 1) * per);
        int c = 0;
#pragma unroll 4
        for (int b = q * per; b < b1; ++b) c += A.hist[(size_t)b * A.experts + e];
        part[i] = c;
    }
    __syncthreads();
    for (int e = tid; e < A.experts; e += 1024) {
        int c = 0;
        for (int q = 0; q < runs; ++q) { const int v = part[q * A.experts + e]; part[q * A.experts + e] = c; c += v; }
        icnt[e] = c;
    }
    __syncthreads();
    ob_route_offsets(A, icnt, scan, tid);
    __syncthreads();
    for (int i = tid; i < runs * A.experts; i += 1024) {
        const int q = i / A.experts, e = i - q * A.experts, b1 = min(n_wg, (q + 1) * per);
        int c = icnt[e] + part[i];
        for (int b = q * per; b < b1; ++b) {
            int *h = A.hist + (size_t)b * A.experts + e;
            const int v = *h;
            *h = c;
            c += v;
        }
    }
}

// third pass: every token's row
__global__ __launch_bounds__(256) void ob_route_rows_kernel(const ObRouteArgs A)
{
    extern __shared__ int icnt[];                                     // [experts]
    const int tid = threadIdx.x, t0 = blockIdx.x * OB_MOE_TOKENS, t1 = min(A.T, t0 + OB_MOE_TOKENS);
    for (int e = tid; e < A.experts; e += 256) icnt[e] = A.hist[(size_t)blockIdx.x * A.experts + e];
    __syncthreads();
    for (int i = t0 * A.top + tid; i < t1 * A.top; i += 256) {
        const int e = A.tok_row[i];
        if (e < 0) continue;
        const int r = atomicAdd(&icnt[e], 1);
        A.gather[r] = i / A.top;
        A.tok_row[i] = r;
    }
}
