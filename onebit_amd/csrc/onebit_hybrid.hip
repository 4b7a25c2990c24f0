// libonebit_hybrid.so: one scheduler step of a hybrid decoder (include/onebit_hybrid.h) -- the token rows of all scheduled items
// concatenated, every matrix product one launch over all rows, mixers per item on its own slot, the output head on the rows that
// sample.  Launches per layer run: norm, input product, mixer (attention decode 1, prompts 2; state space 2, prompts 3), output product.
#include <hip/hip_runtime.h>
#include <algorithm>
#include <mutex>
#include <set>
#include <utility>
#include <stdarg.h>
#include <stdio.h>

#include "../../include/onebit.h"
#include "../../include/onebit_hybrid.h"
#include "ob_dense.h"
#include "ob_hrows.h"
#include "ob_flash.h"
#include "ob_sigattn.h"
#include "ob_ssm.h"

static thread_local char g_err[512];
static int hfail(int code, const char *fmt, ...)
{
    va_list ap;
    va_start(ap, fmt);
    vsnprintf(g_err, sizeof(g_err), fmt, ap);
    va_end(ap);
    return code;
}
static int hstatus(const char *what)
{
    const hipError_t e = hipGetLastError();
    return e == hipSuccess ? 0 : hfail((int)e, "%s: %s", what, hipGetErrorString(e));
}
extern "C" int onebit_hybrid_abi_version(void) { return ONEBIT_HYBRID_ABI_VERSION; }
extern "C" const char *onebit_hybrid_last_error(void) { return g_err; }

static inline int64_t cdiv(int64_t a, int64_t b) { return (a + b - 1) / b; }
static inline int64_t rup(int64_t a, int64_t b) { return cdiv(a, b) * b; }
// more than 64 KB of LDS: allowed once per (device, kernel), up to the 160 KB of a CU
static bool lds_ok(const void *f, int bytes)
{
    if (bytes <= 64 * 1024) return true;
    if (bytes > 160 * 1024) return false;
    static std::mutex mx;
    static std::set<std::pair<int, const void *>> done;
    int dev = 0;
    (void)hipGetDevice(&dev);
    std::lock_guard<std::mutex> g(mx);
    if (done.count({dev, f})) return true;
    if (hipFuncSetAttribute(f, hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024) != hipSuccess) return false;
    done.insert({dev, f});
    return true;
}

// ------------------------------------------------------------------------------------------------------ dense products --
#define OB_SKINNY_T 64
#define OB_ZROWS 2048           // fp32 rows the partial-sum buffer holds at least: splits * T <= max(OB_ZROWS, T)

// K splits of an output product: enough workgroups to fill the chip, each with a worthwhile share of k tiles
static int gemm_splits(int n_tiles, int nkt, int T)
{
    int64_t wgs, min_kt;
    if (T <= OB_SKINNY_T) { wgs = cdiv(n_tiles, 2); min_kt = 16; }
    else { wgs = cdiv(n_tiles, 8) * cdiv(T, 128); min_kt = 16; }
    const int64_t want = T <= OB_SKINNY_T ? 512 : 384;
    int64_t s = std::min<int64_t>({cdiv(want, wgs), std::max<int64_t>(1, nkt / min_kt), std::max(1, OB_ZROWS / T), 8});
    if (T > OB_SKINNY_T && wgs >= 192) s = 1;
    return (int)std::max<int64_t>(1, s);
}

template <typename E, int EPI>
static int dense_launch(ObDenseArgs a, int n_split, hipStream_t s)
{
    if (a.T <= 0 || a.n_tiles <= 0) return 0;
    a.kt_split = (int)cdiv(a.nkt, n_split);
    n_split = (int)cdiv(a.nkt, a.kt_split);               // (no empty split)
    if (a.T <= OB_SKINNY_T) {
        const dim3 grid((unsigned)cdiv(a.n_tiles, 2), (unsigned)n_split);
        if (a.T <= 16) hipLaunchKernelGGL((ob_dense_skinny_kernel<E, EPI, 1>), grid, dim3(256), 0, s, a);
        else if (a.T <= 32) hipLaunchKernelGGL((ob_dense_skinny_kernel<E, EPI, 2>), grid, dim3(256), 0, s, a);
        else hipLaunchKernelGGL((ob_dense_skinny_kernel<E, EPI, 4>), grid, dim3(256), 0, s, a);
        return hstatus("dense product");
    }
    if constexpr (sizeof(E) == 2) {
        if (cdiv(a.n_tiles, 16) * cdiv(a.T, 256) * n_split >= 224) {
            auto k = ob_dense_tile_kernel<E, EPI, 16, 16, 2, 4, 4>;
            const int lds = 4 * 32 * 1024;
            if (!lds_ok((const void *)k, lds)) return hfail(ONEBIT_E_SHAPE, "dense product: LDS");
            hipLaunchKernelGGL(k, dim3((unsigned)(cdiv(a.n_tiles, 16) * cdiv(a.T, 256)), (unsigned)n_split), dim3(512), lds, s, a);
            return hstatus("dense product");
        }
    }
    auto k = ob_dense_tile_kernel<E, EPI, 8, 8, 2, 2, 4>;
    const int lds = 4 * 16 * 1024;
    if (!lds_ok((const void *)k, lds)) return hfail(ONEBIT_E_SHAPE, "dense product: LDS");
    hipLaunchKernelGGL(k, dim3((unsigned)(cdiv(a.n_tiles, 8) * cdiv(a.T, 128)), (unsigned)n_split), dim3(256), lds, s, a);
    return hstatus("dense product");
}

extern "C" int onebit_hybrid_gemm_splits(int32_t n_tiles, int32_t nkt, int32_t T) { return n_tiles > 0 && nkt > 0 && T > 0 ? gemm_splits(n_tiles, nkt, T) : 0; }
extern "C" int onebit_hybrid_gemm(const void *w, const void *a, float *z, int32_t dtype, int32_t n_tiles, int32_t nkt, int32_t T, int32_t n_split, void *stream)
{
    if (!w || !a || !z || n_tiles <= 0 || nkt <= 0 || T < 0 || n_split < 1 || n_split > nkt || nkt % n_split) return hfail(ONEBIT_E_ARG, "hybrid_gemm: bad arguments");
    ObDenseArgs d = {};
    d.w = w; d.a = a; d.n_tiles = n_tiles; d.nkt = nkt; d.T = T;
    d.z = z; d.ldz = 16 * n_tiles; d.z_split = (size_t)T * d.ldz;
    if (dtype == ONEBIT_HYB_BF16) return dense_launch<__bf16, OB_EPI_PART>(d, n_split, (hipStream_t)stream);
    if (dtype == ONEBIT_HYB_F32) return dense_launch<float, OB_EPI_PART>(d, n_split, (hipStream_t)stream);
    return hfail(ONEBIT_E_DTYPE, "hybrid_gemm: dtype %d", dtype);
}

// ----------------------------------------------------------------------------------------------------------- workspace --
struct HPlan {
    size_t x, emb0, h, u, aux, z, qn, xbc, y, part, ticket, out_h, total;
    size_t act[64]; int n_act; int act_mix[64], act_act[64];       // one activation buffer per distinct (mix_k, act_k): its padding stays zero
};
static int act_index(const HPlan &P, const onebit_hlayer_t &L)
{
    for (int i = 0; i < P.n_act; ++i) if (P.act_mix[i] == L.mix_k && P.act_act[i] == L.act_k) return i;
    return -1;
}
static int make_plan(const onebit_hmodel_t &m, int64_t rows, int64_t n_out, int max_dec, int max_splits, HPlan &P)
{
    const size_t es = m.dtype == ONEBIT_HYB_BF16 ? 2 : 4;
    const int64_t R = rup(rows, 256), O = rup(std::max<int64_t>(n_out, 1), 256);
    int64_t u = 0, aux = 0, qn = 0, xbc = 0, y = 0, hd = 0;
    bool loop = false;
    P.n_act = 0;
    size_t o = 0;
    auto take = [&](size_t bytes) { const size_t at = o; o += (bytes + 255) & ~(size_t)255; return at; };
    for (int i = 0; i < m.n_runs; ++i) loop |= m.runs[i].add_embedding != 0;
    for (int i = 0; i < m.n_layers; ++i) {
        const onebit_hlayer_t &L = m.layers[i];
        u = std::max<int64_t>(u, 16LL * L.nt_mix);
        aux = std::max<int64_t>(aux, 16LL * L.nt_aux);
        if (L.kind == ONEBIT_MIX_SIGMOID_ATTENTION) { qn = std::max<int64_t>(qn, (int64_t)L.heads * L.kp); hd = std::max<int64_t>(hd, (int64_t)L.heads * 128); }
        else {
            y = std::max<int64_t>(y, rup((int64_t)L.heads * L.vdim, 8));
            xbc = std::max<int64_t>(xbc, rup((int64_t)L.heads * L.vdim + 2LL * L.groups * L.state, 8));
        }
        if (act_index(P, L) < 0) {
            if (P.n_act == 64) return hfail(ONEBIT_E_SHAPE, "hybrid: more than 64 distinct layer shapes");
            P.act_mix[P.n_act] = L.mix_k; P.act_act[P.n_act] = L.act_k;
            P.act[P.n_act++] = take((size_t)R * (L.mix_k + L.act_k) * es);
        }
    }
    P.x = take((size_t)R * m.width * 4);
    P.emb0 = take(loop ? (size_t)R * m.width * 4 : 0);
    P.h = take((size_t)R * m.width_pad * es);
    P.u = take((size_t)R * u * es);
    P.aux = take((size_t)R * aux * 4);
    P.z = take((size_t)std::max<int64_t>(R, OB_ZROWS) * rup(m.width, 16) * 4);
    P.qn = take((size_t)R * qn * es);
    P.xbc = take((size_t)R * xbc * es);
    P.y = take((size_t)R * y * es);
    P.part = take(max_splits > 1 ? (size_t)max_dec * max_splits * hd * 4 : 0);
    P.ticket = take((size_t)max_dec * hd / 128 * 4);
    P.out_h = take((size_t)O * m.width_pad * es);
    P.total = o;
    return 0;
}

static int check_model(const onebit_hmodel_t *m)
{
    if (!m) return hfail(ONEBIT_E_ARG, "hybrid: null model");
    if (m->struct_size != sizeof(onebit_hmodel_t)) return hfail(ONEBIT_E_ARG, "hybrid: model struct_size %llu, library %zu", (unsigned long long)m->struct_size, sizeof(onebit_hmodel_t));
    if (m->dtype != ONEBIT_HYB_BF16 && m->dtype != ONEBIT_HYB_F32) return hfail(ONEBIT_E_DTYPE, "hybrid: dtype %d", m->dtype);
    const int kt = m->dtype == ONEBIT_HYB_BF16 ? 32 : 16;
    if (m->width <= 0 || m->width_pad < m->width || m->width_pad % kt || m->vocab <= 0 || m->n_layers <= 0 || m->n_runs < 0 || m->n_slots <= 0 || m->max_len <= 0)
        return hfail(ONEBIT_E_SHAPE, "hybrid: model sizes");
    if (m->width > 32768) return hfail(ONEBIT_E_SHAPE, "hybrid: width %d (at most 32768)", m->width);
    if (m->pos_embed && m->max_len > m->max_pos) return hfail(ONEBIT_E_SHAPE, "hybrid: max_len %d beyond the %d learned positions", m->max_len, m->max_pos);
    if (!m->layers || (m->n_runs && !m->runs) || !m->embed || !m->final_norm || !m->head) return hfail(ONEBIT_E_ARG, "hybrid: null model pointer");
    for (int i = 0; i < m->n_layers; ++i) {
        const onebit_hlayer_t &L = m->layers[i];
        const bool att = L.kind == ONEBIT_MIX_SIGMOID_ATTENTION;
        if (!att && L.kind != ONEBIT_MIX_SSM) return hfail(ONEBIT_E_ARG, "hybrid: layer %d: mixer kind %d", i, L.kind);
        if (!L.w_in || !L.w_out || !L.norm_w || L.heads <= 0 || L.vdim <= 0 || L.nt_mix <= 0 || L.nt_aux < 0 || ((L.nt_mix + L.nt_aux) & 1) ||
            L.nt_in < L.nt_mix + L.nt_aux || ((L.nt_in - L.nt_mix - L.nt_aux) & 1) || L.mix_k % kt || L.act_k % kt || L.mix_k < L.heads * L.vdim ||
            L.act_k < (L.nt_in - L.nt_mix - L.nt_aux) * 8)
            return hfail(ONEBIT_E_SHAPE, "hybrid: layer %d: sizes", i);
        if (att) {
            if (L.kv_heads <= 0 || L.heads % L.kv_heads || L.dim <= 0 || L.dim > 4096 || L.kp < L.dim || L.vp < L.vdim || (L.kp & 7) || (L.vp & 7) ||
                16LL * L.nt_mix < (int64_t)(L.heads + L.kv_heads) * L.dim + (int64_t)L.kv_heads * L.vdim || (L.r1 && !L.r2))
                return hfail(ONEBIT_E_SHAPE, "hybrid: layer %d: attention sizes", i);
            if ((int64_t)m->max_len * std::max(L.kp, L.vp) * 4 > 0x7fffffffLL) return hfail(ONEBIT_E_SHAPE, "hybrid: layer %d: max_len too large", i);
        } else {
            if (L.groups <= 0 || L.heads % L.groups || L.state <= 0 || L.state > 512 || L.taps <= 0 || L.norm_groups <= 0 || (L.heads * L.vdim) % L.norm_groups ||
                L.sp < L.vdim || (L.sp & 3) || 16LL * L.nt_mix < 2LL * L.heads * L.vdim + 2LL * L.groups * L.state || 16 * L.nt_aux < L.heads ||
                !L.conv_w || !L.conv_b || !L.dt_bias || !L.A_log || !L.D || !L.gnorm_w)
                return hfail(ONEBIT_E_SHAPE, "hybrid: layer %d: state-space sizes (state at most 512)", i);
        }
    }
    for (int i = 0; i < m->n_runs; ++i)
        if (m->runs[i].layer < 0 || m->runs[i].layer >= m->n_layers || !m->runs[i].s0 || !m->runs[i].s1) return hfail(ONEBIT_E_ARG, "hybrid: run %d", i);
    return 0;
}

extern "C" size_t onebit_hybrid_workspace_bytes(const onebit_hmodel_t *m, int64_t max_rows, int64_t max_out, int32_t max_dec, int32_t max_splits)
{
    HPlan P;
    if (check_model(m) || max_rows <= 0 || max_dec < 0 || max_splits < 1 || make_plan(*m, max_rows, max_out, max_dec, max_splits, P)) return 0;
    return P.total;
}

// ---------------------------------------------------------------------------------------------------------------- step --
template <typename E>
static int norm_launch(const ObHNormArgs &a, int rows, hipStream_t s)
{
    if (rows <= 0) return 0;
    const int lds = (((a.W + 3) & ~3) + 16) * 4;
    auto k4 = ob_hnorm_kernel<E, 4>;
    auto k1 = ob_hnorm_kernel<E, 1>;
    if (!lds_ok(a.W % 4 == 0 ? (const void *)k4 : (const void *)k1, lds)) return hfail(ONEBIT_E_SHAPE, "norm: LDS");
    const unsigned thr = (unsigned)std::min<int64_t>(rows <= 256 ? 1024 : 512, std::max<int64_t>(64, rup(cdiv(a.W, 4), 64)));
    if (a.W % 4 == 0) hipLaunchKernelGGL(k4, dim3((unsigned)rows), dim3(thr), lds, s, a);
    else hipLaunchKernelGGL(k1, dim3((unsigned)rows), dim3(thr), lds, s, a);
    return hstatus("norm");
}

template <typename E>
static int attention_launch(const onebit_hmodel_t &m, const onebit_hlayer_t &L, const onebit_hrun_t &run, const onebit_hstate_t &st, const HPlan &P,
                            char *ws, void *act, int act_nkt, hipStream_t s)
{
    const bool mfma = sizeof(E) == 2 && L.kp == L.vp && (L.kp == 64 || L.kp == 128);
    const int n_dec = mfma ? st.n_dec : 0, ldu = 16 * L.nt_mix;      // without the tiled forms every row takes the row kernel
    if (n_dec) {
        ObSigDecArgs a = {ws + P.u, ldu, 0, run.s0, run.s1, act, act_nkt, st.row_slot, st.row_pos, L.heads, L.kv_heads, L.dim, L.vdim, m.n_slots, m.max_len,
                          st.attn_chunk, st.attn_splits, L.scale, m.eps, {L.r1, L.r2, L.pb}, L.unit_rms, (float *)(ws + P.part), (int *)(ws + P.ticket)};
        const int rep = L.heads / L.kv_heads, R = rep >= 4 ? 4 : rep >= 2 ? 2 : 1;
        const dim3 grid((unsigned)(L.kv_heads * cdiv(rep, R)), (unsigned)n_dec, (unsigned)st.attn_splits);
#define OB_DEC(DP, R_) hipLaunchKernelGGL((ob_sig_dec_kernel<DP, R_>), grid, dim3(256), 0, s, a)
        if (L.kp == 64) { if (R == 4) OB_DEC(64, 4); else if (R == 2) OB_DEC(64, 2); else OB_DEC(64, 1); }
        else { if (R == 4) OB_DEC(128, 4); else if (R == 2) OB_DEC(128, 2); else OB_DEC(128, 1); }
#undef OB_DEC
        if (int rc = hstatus("decode attention")) return rc;
    }
    const int rest = st.n_rows - n_dec;
    if (!rest) return 0;
    const ObSigPrepArgs p = {ws + P.u, ldu, n_dec, ws + P.qn, run.s0, run.s1, st.row_slot, st.row_pos, rest, L.heads, L.kv_heads, L.dim, L.vdim, L.kp, L.vp,
                             m.n_slots, m.max_len, m.eps, L.unit_rms};
    for (int r0 = 0; r0 < rest; r0 += 32768) {                       // (grid y limit)
        ObSigPrepArgs pp = p;
        pp.row0 = n_dec + r0;
        if constexpr (sizeof(E) == 2) {
            if (mfma && L.dim % 8 == 0 && L.vdim % 8 == 0) {
                const dim3 grid((unsigned)cdiv((int64_t)(L.heads + 2 * L.kv_heads) * (L.kp / 8), 256), (unsigned)std::min(rest - r0, 32768));
                if (L.kp == 64) hipLaunchKernelGGL((ob_sig_prep_vec_kernel<64>), grid, dim3(256), 0, s, pp);
                else hipLaunchKernelGGL((ob_sig_prep_vec_kernel<128>), grid, dim3(256), 0, s, pp);
                continue;
            }
        }
        hipLaunchKernelGGL((ob_sig_prep_kernel<E>), dim3((unsigned)cdiv(L.heads + 2 * L.kv_heads, 4), (unsigned)std::min(rest - r0, 32768)), dim3(256), 0, s, pp);
    }
    if (int rc = hstatus("attention inputs")) return rc;
    if (!mfma) {
        for (int r0 = 0; r0 < rest; r0 += 32768) {
            const ObSigRowsArgs a = {ws + P.qn, run.s0, run.s1, act, act_nkt, st.row_slot, st.row_pos, n_dec + r0, L.heads, L.kv_heads, L.dim, L.vdim, L.kp, L.vp,
                                     m.n_slots, m.max_len, L.scale, {L.r1, L.r2, L.pb}};
            hipLaunchKernelGGL((ob_sig_rows_kernel<E>), dim3((unsigned)L.heads, (unsigned)std::min(rest - r0, 32768)), dim3(256), L.dim * 4, s, a);
        }
        return hstatus("attention rows");
    }
    for (int s0 = 0; s0 < st.n_seg; s0 += OB_FL_MAXSEG) {
        const int ns = std::min(st.n_seg - s0, OB_FL_MAXSEG);
        ObFlashSigArgs a = {};
        a.a.q = (const _Float16 *)(ws + P.qn); a.a.k = (const _Float16 *)run.s0; a.a.v = (const _Float16 *)run.s1;      // (bf16 behind these pointers)
        a.a.H = L.heads; a.a.Hkv = L.kv_heads; a.a.max_len = m.max_len;
        a.a.scale_log2e = -L.scale * OB_LOG2E;
        a.r1 = L.r1; a.r2 = L.r2; a.pb = L.pb; a.out = act; a.out_nkt = act_nkt; a.vdim = L.vdim;
        a.nseg = ns;
        int64_t wgs = 0;
        for (int i = 0; i < ns; ++i) {
            const onebit_hseg_t &g = st.segs[s0 + i];
            const int64_t nmb = cdiv(g.n, OB_FL_BM);
            wgs += (nmb + 1) / 2 * L.heads;
            if (wgs > 0x3fffffffLL) return hfail(ONEBIT_E_ARG, "attention: too many workgroups");
            a.wg_end[i] = (int)wgs;
            a.seg[i] = {g.row0, g.n, g.slot, g.past};
        }
        if (L.kp == 128) hipLaunchKernelGGL((ob_flash_fwd_kernel<128, true, ObFlSigmoidBf16>), dim3((unsigned)wgs), dim3(256), 0, s, a);
        else hipLaunchKernelGGL((ob_flash_fwd_kernel<64, true, ObFlSigmoidBf16>), dim3((unsigned)wgs), dim3(256), 0, s, a);
    }
    return hstatus("prompt attention");
}

template <typename E>
static int ssm_launch(const onebit_hmodel_t &m, const onebit_hlayer_t &L, const onebit_hrun_t &run, const onebit_hstate_t &st, const HPlan &P, char *ws,
                      void *act, int act_nkt, hipStream_t s)
{
    constexpr int VEC = ObElem<E>::EPL;
    const int inner = L.heads * L.vdim, ch = inner + 2 * L.groups * L.state, ldy = (int)rup(inner, 8), ldx = (int)rup(ch, 8), nsl = (int)cdiv(L.vdim, 32);
    ObSsmArgs a = {ws + P.u, 16 * L.nt_mix, inner, nullptr, ldx, (const float *)(ws + P.aux), 16 * L.nt_aux, L.conv_w, L.conv_b, L.dt_bias, L.A_log, L.D,
                   (float *)run.s0, run.s1, ws + P.y, ldy, st.row_slot, st.row_pos, 0, L.heads, L.groups, L.state, L.vdim, L.sp, L.taps, ch, m.n_slots, m.max_len};
    auto step = [&](const ObSsmArgs &aa, const ObSsmSegs &sg, int n) {
        const dim3 grid((unsigned)(L.heads * nsl), (unsigned)n);
        if (L.state <= 64) hipLaunchKernelGGL((ob_ssm_step_kernel<E, 2>), grid, dim3(256), 0, s, aa, sg);
        else if (L.state <= 128) hipLaunchKernelGGL((ob_ssm_step_kernel<E, 4>), grid, dim3(256), 0, s, aa, sg);
        else if (L.state <= 256) hipLaunchKernelGGL((ob_ssm_step_kernel<E, 8>), grid, dim3(256), 0, s, aa, sg);
        else hipLaunchKernelGGL((ob_ssm_step_kernel<E, 16>), grid, dim3(256), 0, s, aa, sg);
    };
    if (st.n_dec) {
        step(a, ObSsmSegs{}, st.n_dec);
        if (int rc = hstatus("state-space decode")) return rc;
    }
    if (st.n_seg) {
        const int rest = st.n_rows - st.n_dec;
        a.xbc = ws + P.xbc;
        for (int r0 = 0; r0 < rest; r0 += 32768) {
            ObSsmArgs c = a;
            c.row0 = st.n_dec + r0;
            const unsigned ny = (unsigned)std::min(rest - r0, 32768);
            if (ch % VEC == 0 && inner % VEC == 0 && L.taps >= 2 && L.taps <= 4) {
                const dim3 grid((unsigned)cdiv(ch / VEC, 256), (unsigned)cdiv(ny, OB_CONV_ROWS));
                const int last = st.n_dec + r0 + (int)ny;
                if (L.taps == 2) hipLaunchKernelGGL((ob_conv_rows_kernel<E, 2>), grid, dim3(256), 0, s, c, st.row_off, ws + P.xbc, last);
                else if (L.taps == 3) hipLaunchKernelGGL((ob_conv_rows_kernel<E, 3>), grid, dim3(256), 0, s, c, st.row_off, ws + P.xbc, last);
                else hipLaunchKernelGGL((ob_conv_rows_kernel<E, 4>), grid, dim3(256), 0, s, c, st.row_off, ws + P.xbc, last);
            } else if (ch % VEC == 0 && inner % VEC == 0) hipLaunchKernelGGL((ob_conv_kernel<E, VEC>), dim3((unsigned)cdiv(ch / VEC, 256), ny), dim3(256), 0, s, c, st.row_off, ws + P.xbc);
            else hipLaunchKernelGGL((ob_conv_kernel<E, 1>), dim3((unsigned)cdiv(ch, 256), ny), dim3(256), 0, s, c, st.row_off, ws + P.xbc);
        }
        if (int rc = hstatus("convolution")) return rc;
        for (int s0 = 0; s0 < st.n_seg; s0 += OB_SSM_MAXSEG) {
            ObSsmSegs sg = {};
            sg.nseg = std::min(st.n_seg - s0, OB_SSM_MAXSEG);
            for (int i = 0; i < sg.nseg; ++i) { const onebit_hseg_t &g = st.segs[s0 + i]; sg.s[i] = {g.row0, g.n, g.slot, g.past}; }
            bool done = false;
            if constexpr (sizeof(E) == 2) {
                const bool vec = L.state % 8 == 0 && L.vdim % 8 == 0;
                const dim3 grid((unsigned)(L.heads * nsl), (unsigned)sg.nseg);
#define OB_SSD(NP) do { if (vec) hipLaunchKernelGGL((ob_ssd_kernel<NP, true>), grid, dim3(256), 0, s, a, sg); \
                        else hipLaunchKernelGGL((ob_ssd_kernel<NP, false>), grid, dim3(256), 0, s, a, sg); done = true; } while (0)
                if (L.state <= 64) OB_SSD(64);
                else if (L.state <= 128) OB_SSD(128);
                else if (L.state <= 256) OB_SSD(256);
#undef OB_SSD
            }
            if (!done) step(a, sg, sg.nseg);
            if (int rc = hstatus("state-space scan")) return rc;
        }
    }
    ObGatedNormArgs n = {ws + P.y, ldy, ws + P.u, 16 * L.nt_mix, L.gnorm_w, m.eps, inner / L.norm_groups, act, act_nkt};
    const int lds = (((n.gsize + 3) & ~3) + 16) * 4;
    auto k4 = ob_gated_norm_kernel<E, VEC>;
    auto k1 = ob_gated_norm_kernel<E, 1>;
    if (!lds_ok(n.gsize % VEC == 0 ? (const void *)k4 : (const void *)k1, lds)) return hfail(ONEBIT_E_SHAPE, "gated norm: LDS");
    for (int r0 = 0; r0 < st.n_rows; r0 += 32768) {
        // (32768 rows = a whole number of 16-row bands: the fragment-major rows of the slice start at a band)
        n.y = ws + P.y + (size_t)r0 * ldy * sizeof(E);
        n.gate = ws + P.u + (size_t)r0 * n.ldg * sizeof(E);
        n.out = (char *)act + (size_t)(r0 / 16) * act_nkt * 1024;
        const dim3 grid((unsigned)L.norm_groups, (unsigned)std::min(st.n_rows - r0, 32768));
        const unsigned thr = (unsigned)std::min<int64_t>(256, std::max<int64_t>(64, rup(cdiv(n.gsize, VEC), 64)));
        if (n.gsize % VEC == 0) hipLaunchKernelGGL(k4, grid, dim3(thr), lds, s, n);
        else hipLaunchKernelGGL(k1, grid, dim3(256), lds, s, n);
    }
    return hstatus("gated norm");
}

template <typename E>
static int step_impl(const onebit_hmodel_t &m, const onebit_hstate_t &st, const HPlan &P, hipStream_t s)
{
    constexpr int KT = ObElem<E>::KT;
    char *ws = (char *)st.workspace;
    const int T = st.n_rows, ldz = (int)rup(m.width, 16), w_nkt = m.width_pad / KT;
    ObHNormArgs nb = {};
    nb.x = (float *)(ws + P.x); nb.ldz = ldz; nb.mult = m.mult; nb.off = m.norm_off; nb.eps = m.eps; nb.W = m.width; nb.out_nkt = w_nkt;
    nb.tokens = st.tokens; nb.row_pos = st.row_pos;
    bool loop = false;
    for (int i = 0; i < m.n_runs; ++i) loop |= m.runs[i].add_embedding != 0;
    // what the next row kernel adds to the residual: nothing yet (the embedding), or the last output product
    ObHNormArgs pend = nb;
    pend.embed = m.embed; pend.pos_embed = m.pos_embed;
    if (loop) pend.emb_save = (float *)(ws + P.emb0);
    auto residual_out = [&](int run) -> int {      // x + (pending product), without touching the stream's own copy
        if (!st.residuals) return 0;
        float *dst = st.residuals + (size_t)run * T * m.width;
        const hipError_t e = hipMemcpyAsync(dst, ws + P.x, (size_t)T * m.width * 4, hipMemcpyDeviceToDevice, s);
        if (e != hipSuccess) return hfail((int)e, "residual copy: %s", hipGetErrorString(e));
        ObHNormArgs a = pend;
        a.x = dst; a.w = m.final_norm; a.out = ws + P.out_h;      // (norm output unused; see the size check in onebit_hybrid_step)
        a.emb_save = nullptr;
        return norm_launch<E>(a, T, s);
    };
    for (int r = 0; r < m.n_runs; ++r) {
        const onebit_hrun_t &run = m.runs[r];
        const onebit_hlayer_t &L = m.layers[run.layer];
        const int ai = act_index(P, L), act_nkt = (L.mix_k + L.act_k) / KT;
        void *act = ws + P.act[ai];
        ObHNormArgs a = pend;
        a.w = L.norm_w; a.out = ws + P.h;
        if (run.add_embedding) a.emb_add = (const float *)(ws + P.emb0);
        if (int rc = norm_launch<E>(a, T, s)) return rc;
        ObDenseArgs d = {};
        d.w = L.w_in; d.a = ws + P.h; d.n_tiles = L.nt_in; d.nkt = w_nkt; d.T = T;
        d.bias = L.b_in; d.u = ws + P.u; d.nt_mix = L.nt_mix; d.aux = (float *)(ws + P.aux); d.nt_aux = L.nt_aux;
        d.act = act; d.act_k0 = L.mix_k; d.act_nkt = act_nkt;
        if (int rc = dense_launch<E, OB_EPI_IN>(d, 1, s)) return rc;
        const int rc = L.kind == ONEBIT_MIX_SIGMOID_ATTENTION ? attention_launch<E>(m, L, run, st, P, ws, act, act_nkt, s)
                                                              : ssm_launch<E>(m, L, run, st, P, ws, act, act_nkt, s);
        if (rc) return rc;
        ObDenseArgs o = {};
        o.w = L.w_out; o.a = act; o.n_tiles = ldz / 16; o.nkt = act_nkt; o.T = T;
        o.z = (float *)(ws + P.z); o.ldz = ldz; o.z_split = (size_t)T * ldz;
        int n_split = gemm_splits(o.n_tiles, o.nkt, T);
        n_split = (int)cdiv(o.nkt, cdiv(o.nkt, n_split));
        if (int rc2 = dense_launch<E, OB_EPI_PART>(o, n_split, s)) return rc2;
        pend = nb;
        pend.z = o.z; pend.z_split = o.z_split; pend.n_split = n_split; pend.bias = L.b_out;
        if (int rc2 = residual_out(r)) return rc2;
    }
    if (st.n_out > 0) {
        ObHNormArgs a = pend;
        a.w = m.final_norm; a.out = ws + P.out_h; a.rows = st.out_rows; a.emb_save = nullptr;
        if (int rc = norm_launch<E>(a, st.n_out, s)) return rc;
        ObDenseArgs d = {};
        d.w = m.head; d.a = ws + P.out_h; d.n_tiles = (int)cdiv(m.vocab, 16); d.nkt = w_nkt; d.T = st.n_out;
        d.logits = st.logits; d.V = m.vocab; d.cap = m.softcap;
        if (int rc = dense_launch<E, OB_EPI_LOGITS>(d, 1, s)) return rc;
        if (st.next_tokens) {
            hipLaunchKernelGGL(ob_argmax_rows_kernel, dim3((unsigned)st.n_out), dim3(1024), 0, s, st.logits, st.next_tokens, m.vocab);
            return hstatus("argmax");
        }
    }
    return 0;
}

extern "C" int onebit_hybrid_step(const onebit_hmodel_t *m, const onebit_hstate_t *st, int64_t max_rows, int64_t max_out, int32_t max_dec, int32_t max_splits,
                                  void *stream)
{
    if (int rc = check_model(m)) return rc;
    if (!st) return hfail(ONEBIT_E_ARG, "hybrid_step: null state");
    if (st->struct_size != sizeof(onebit_hstate_t)) return hfail(ONEBIT_E_ARG, "hybrid_step: state struct_size %llu, library %zu", (unsigned long long)st->struct_size, sizeof(onebit_hstate_t));
    if (st->n_rows < 0 || st->n_dec < 0 || st->n_seg < 0 || st->n_out < 0 || st->n_dec > st->n_rows) return hfail(ONEBIT_E_ARG, "hybrid_step: negative size");
    if (st->n_rows == 0) return 0;
    if (st->n_rows > max_rows || st->n_out > max_out || st->n_dec > max_dec || st->attn_splits > max_splits) return hfail(ONEBIT_E_SHAPE, "hybrid_step: step larger than its workspace");
    if (!st->tokens || !st->row_slot || !st->row_pos || !st->row_off || (st->n_seg && !st->segs) || (st->n_out && (!st->out_rows || !st->logits)) || !st->workspace)
        return hfail(ONEBIT_E_ARG, "hybrid_step: null pointer");
    if (st->n_dec && (st->attn_splits < 1 || st->attn_chunk < 128 || st->attn_chunk % 128)) return hfail(ONEBIT_E_SHAPE, "hybrid_step: attn_chunk must be a multiple of 128");
    if (st->residuals && st->n_rows > rup(std::max<int64_t>(max_out, 1), 256)) return hfail(ONEBIT_E_SHAPE, "hybrid_step: residuals need room for n_rows output rows");
    int row = st->n_dec;
    for (int i = 0; i < st->n_seg; ++i) {
        const onebit_hseg_t &g = st->segs[i];
        if (g.row0 != row || g.n < 1 || g.slot < 0 || g.slot >= m->n_slots || g.past < 0 || (int64_t)g.past + g.n > m->max_len)
            return hfail(ONEBIT_E_SHAPE, "hybrid_step: segment %d (rows %d + %d, slot %d, past %d)", i, g.row0, g.n, g.slot, g.past);
        row += g.n;
    }
    if (row != st->n_rows) return hfail(ONEBIT_E_SHAPE, "hybrid_step: n_rows %d, decode rows and segments make %d", st->n_rows, row);
    HPlan P;
    if (int rc = make_plan(*m, max_rows, max_out, max_dec, max_splits, P)) return rc;
    if (st->workspace_bytes < P.total || ((uintptr_t)st->workspace & 255)) return hfail(ONEBIT_E_WSPACE, "hybrid_step: workspace %zu of %zu bytes (256-byte aligned)", st->workspace_bytes, P.total);
    return m->dtype == ONEBIT_HYB_BF16 ? step_impl<__bf16>(*m, *st, P, (hipStream_t)stream) : step_impl<float>(*m, *st, P, (hipStream_t)stream);
}
