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
static inline size_t ob_route_lds(const ObRouteArgs &A) { return ((size_t)16 * (A.experts + A.identity) + 16 * A.groups) * 4 + (size_t)A.experts * 4; }

// one wave per token: choice scores in LDS, every lane ranks its own entries against all others
__device__ __forceinline__ void ob_route_token(const ObRouteArgs &A, int t, float *cs, float *gs, int lane)
{
    const int N = A.experts + A.identity, per = N / A.groups;
    const float *z = A.z + (size_t)t * A.ldz;
    float mx = -INFINITY;
    for (int i = lane; i < N; i += 64) mx = fmaxf(mx, z[i]);
    mx = ob_wave_max(mx);
    float sum = 0.f;
    for (int i = lane; i < N; i += 64) sum += expf(z[i] - mx);
    sum = ob_wave_sum(sum);
    auto score = [&](int i) { return expf(z[i] - mx) / sum; };
    for (int i = lane; i < N; i += 64) cs[i] = score(i) + A.correction[i];
    for (int k = lane; k < A.top; k += 64) { A.tok_row[(size_t)t * A.top + k] = -1; A.tok_w[(size_t)t * A.top + k] = 0.f; }
    __builtin_amdgcn_wave_barrier();
    asm volatile("s_waitcnt vmcnt(0) lgkmcnt(0)" ::: "memory");       // (this wave's LDS and the cleared slots)
    if (A.keep < A.groups) {
        for (int g = lane; g < A.groups; g += 64) {
            float m = -INFINITY;
            for (int i = 0; i < per; ++i) m = fmaxf(m, cs[g * per + i]);
            gs[g] = m;
        }
        __builtin_amdgcn_wave_barrier();
        asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
    }
    auto allowed = [&](int i) {
        if (A.keep >= A.groups) return true;
        const int g = i / per;
        int r = 0;
        for (int o = 0; o < A.groups; ++o) r += gs[o] > gs[g] || (gs[o] == gs[g] && o < g);
        return r < A.keep;
    };
    for (int i = lane; i < N; i += 64) if (!allowed(i)) cs[i] = -INFINITY;
    __builtin_amdgcn_wave_barrier();
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
    float idw = 0.f;
    for (int i = lane; i < N; i += 64) {
        const float c = cs[i];
        if (c == -INFINITY) continue;
        int r = 0;
        for (int o = 0; o < N; ++o) r += cs[o] > c || (cs[o] == c && o < i);
        if (r >= A.top) continue;
        const float w = score(i);
        if (i >= A.experts) idw += w;
        else { A.tok_row[(size_t)t * A.top + r] = i; A.tok_w[(size_t)t * A.top + r] = w; }
    }
    idw = ob_wave_sum(idw);
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
template <bool SINGLE>
__global__ __launch_bounds__(1024) void ob_route_kernel(const ObRouteArgs A)
{
    extern __shared__ __attribute__((aligned(16))) float sm[];        // [16][N] choices | [16][groups] | [experts] counts
    __shared__ int scan[32];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, N = A.experts + A.identity;
    float *cs = sm + (size_t)wave * N, *gs = sm + (size_t)16 * N + wave * A.groups;
    int *cnt = reinterpret_cast<int *>(sm + (size_t)16 * N + 16 * A.groups);
    for (int e = tid; e < A.experts; e += 1024) cnt[e] = 0;
    const int t0 = blockIdx.x * OB_MOE_TOKENS, t1 = min(A.T, t0 + OB_MOE_TOKENS);
    for (int t = t0 + wave; t < t1; t += 16) {
        ob_route_token(A, t, cs, gs, lane);
        __builtin_amdgcn_wave_barrier();
    }
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    __syncthreads();                                                  // (the slots are read back by other lanes of this workgroup: same CU)
    for (int i = t0 * A.top + tid; i < t1 * A.top; i += 1024) {
        const int e = __hip_atomic_load(A.tok_row + i, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_WORKGROUP);
        if (e >= 0) atomicAdd(&cnt[e], 1);
    }
    __syncthreads();
    if constexpr (!SINGLE) {
        for (int e = tid; e < A.experts; e += 1024) A.hist[(size_t)blockIdx.x * A.experts + e] = cnt[e];
    } else {
        ob_route_offsets(A, cnt, scan, tid);
        __syncthreads();
        for (int i = tid; i < A.T * A.top; i += 1024) {
            const int e = __hip_atomic_load(A.tok_row + i, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_WORKGROUP);
            if (e < 0) continue;
            const int r = atomicAdd(&cnt[e], 1);                      // (the order within an expert is free: every row is computed alone)
            A.gather[r] = i / A.top;
            A.tok_row[i] = r;
        }
    }
}

// second pass, one workgroup: counts of all workgroups -> where each workgroup's tokens of an expert start; row and block tables
__global__ __launch_bounds__(1024) void ob_route_scan_kernel(const ObRouteArgs A, int n_wg)
{
    extern __shared__ int icnt[];                                     // [experts]
    __shared__ int scan[32];
    const int tid = threadIdx.x;
    for (int e = tid; e < A.experts; e += 1024) {
        int c = 0;
        for (int b = 0; b < n_wg; b += 8) {
            int v[8];
#pragma unroll
            for (int j = 0; j < 8; ++j) v[j] = A.hist[(size_t)min(b + j, n_wg - 1) * A.experts + e];
#pragma unroll
            for (int j = 0; j < 8; ++j)
                if (b + j < n_wg) { A.hist[(size_t)(b + j) * A.experts + e] = c; c += v[j]; }
        }
        icnt[e] = c;
    }
    __syncthreads();
    ob_route_offsets(A, icnt, scan, tid);
    __syncthreads();
    for (int e = tid; e < A.experts; e += 1024) {
        const int r0 = icnt[e];
        for (int b = 0; b < n_wg; ++b) A.hist[(size_t)b * A.experts + e] += r0;
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
