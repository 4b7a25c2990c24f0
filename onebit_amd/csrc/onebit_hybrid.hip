// libonebit_hybrid.so: one scheduler step of a hybrid decoder (include/onebit_hybrid.h) -- the token rows of all scheduled items
// concatenated, every matrix product one launch over all rows, mixers per item on its own slot, the output head on the rows that
// sample.  Launches per parallel layer run: norm, input product, mixer (attention decode 1, prompts 2; state space 2, prompts 3), output
// product.  Sequential layers: row kernel, mixer, row kernel, feed-forward (and row kernel, token input); a row kernel finishes the sublayer
// before it (sums, output norm, residual, depth average) and forms the input of the next.
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
#include "ob_latent.h"
#include "ob_moe.h"

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

// few rows, block-diagonal over heads (row-major activations), 64 rows at a time.  `out_step`: bytes of 64 output rows.
template <typename E, int EPI>
static int dense_heads_launch(ObDenseArgs a, size_t out_step, hipStream_t s)
{
    a.kt_split = a.nkt;
    const dim3 grid((unsigned)cdiv(a.n_tiles, 2));
    for (int T = a.T; T > 0; T -= OB_SKINNY_T) {
        a.T = std::min(T, OB_SKINNY_T);
        if (a.T <= 16) hipLaunchKernelGGL((ob_dense_skinny_kernel<E, EPI, 1, OB_ROWS_HEADS>), grid, dim3(256), 0, s, a);
        else if (a.T <= 32) hipLaunchKernelGGL((ob_dense_skinny_kernel<E, EPI, 2, OB_ROWS_HEADS>), grid, dim3(256), 0, s, a);
        else hipLaunchKernelGGL((ob_dense_skinny_kernel<E, EPI, 4, OB_ROWS_HEADS>), grid, dim3(256), 0, s, a);
        a.a = (const char *)a.a + (size_t)OB_SKINNY_T * a.lda * sizeof(E);
        a.u = (char *)a.u + out_step;
        a.act = (char *)a.act + out_step;
        a.heads = (char *)a.heads + out_step;
    }
    return hstatus("per-head product");
}

// the rows of experts: n_blk blocks of at most block_rows (64: few rows; 128 / 256: tiles)
template <typename E, int EPI, int ROWS>
static int dense_blocks_launch(ObDenseArgs a, int n_blk, int block_rows, int n_split, hipStream_t s)
{
    a.kt_split = (int)cdiv(a.nkt, n_split);
    n_split = (int)cdiv(a.nkt, a.kt_split);
    if (block_rows <= OB_SKINNY_T) {
        const dim3 grid((unsigned)cdiv(a.n_tiles, 2), (unsigned)n_split, (unsigned)n_blk);
        if (a.T <= 16) hipLaunchKernelGGL((ob_dense_skinny_kernel<E, EPI, 1, ROWS>), grid, dim3(256), 0, s, a);
        else if (a.T <= 32) hipLaunchKernelGGL((ob_dense_skinny_kernel<E, EPI, 2, ROWS>), grid, dim3(256), 0, s, a);
        else hipLaunchKernelGGL((ob_dense_skinny_kernel<E, EPI, 4, ROWS>), grid, dim3(256), 0, s, a);
        return hstatus("expert product");
    }
    a.T = n_blk * block_rows;
    if constexpr (sizeof(E) == 2) {
        if (block_rows == 256) {
            auto k = ob_dense_tile_kernel<E, EPI, 16, 16, 2, 4, 4, ROWS>;
            const int lds = 4 * 32 * 1024;
            if (!lds_ok((const void *)k, lds)) return hfail(ONEBIT_E_SHAPE, "expert product: LDS");
            hipLaunchKernelGGL(k, dim3((unsigned)(cdiv(a.n_tiles, 16) * n_blk), (unsigned)n_split), dim3(512), lds, s, a);
            return hstatus("expert product");
        }
    }
    auto k = ob_dense_tile_kernel<E, EPI, 8, 8, 2, 2, 4, ROWS>;
    const int lds = 4 * 16 * 1024;
    if (!lds_ok((const void *)k, lds)) return hfail(ONEBIT_E_SHAPE, "expert product: LDS");
    hipLaunchKernelGGL(k, dim3((unsigned)(cdiv(a.n_tiles, 8) * n_blk), (unsigned)n_split), dim3(256), lds, s, a);
    return hstatus("expert product");
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
    size_t hist, hrm, cq, qu, qa, ctx, lml, kv, actm, actf, acte, acts, spre, ez, route;
    int64_t kv_rows, ez_rows;
    size_t act[64]; int n_act; int act_mix[64], act_act[64];       // one activation buffer per distinct (mix_k, act_k): its padding stays zero
};
static int act_index(const HPlan &P, const onebit_hlayer_t &L)
{
    for (int i = 0; i < P.n_act; ++i) if (P.act_mix[i] == L.mix_k && P.act_act[i] == L.act_k) return i;
    return -1;
}
#define OB_LAT_PARTS 1024       // (row, split) pairs of the latent decode attention with more than one split
#define OB_SIDE_SPLITS 4        // K splits of a token input's gate product
#define OB_EZ_ROWS 4096         // fp32 rows of the experts' partial sums at least
// rows of the experts' sorted space: every (token, choice), each expert's first row at a multiple of 16
static int64_t expert_rows(const onebit_hff_t &f, int64_t T) { return T * f.top + 16 * std::min<int64_t>(f.experts, T * f.top); }
// rows that the absorbed form of latent attention may serve
static int64_t absorbed_rows(const onebit_hlatent_t &l, int64_t rows, int64_t max_dec) { return l.tiled && l.flash ? std::min(rows, max_dec * ONEBIT_HYB_SHORT) : rows; }
static int make_plan(const onebit_hmodel_t &m, int64_t rows, int64_t n_out, int max_dec, int max_splits, HPlan &P)
{
    const size_t es = m.dtype == ONEBIT_HYB_BF16 ? 2 : 4;
    const int64_t R = rup(rows, 256), O = rup(std::max<int64_t>(n_out, 1), 256);
    int64_t u = 0, aux = 0, qn = 0, xbc = 0, y = 0, hd = 0;
    bool loop = false, hist = false, rm = false;
    int64_t cq = 0, qu = 0, qa = 0, lp = 0, lml = 0, kv = 0, am = 0, af = 0, ae = 0, as = 0, ez = 0, rt = 0, zc = rup(m.width, 16);
    const int kt = es == 2 ? 32 : 16;
    P.kv_rows = rup(std::max<int64_t>(m.max_len, rows + 16 * OB_DENSE_MAXSEG), 16);
    P.ez_rows = 0;
    P.n_act = 0;
    size_t o = 0;
    auto take = [&](size_t bytes) { const size_t at = o; o += (bytes + 255) & ~(size_t)255; return at; };
    for (int i = 0; i < m.n_runs; ++i) loop |= m.runs[i].add_embedding != 0;
    for (int i = 0; i < m.n_layers; ++i) {
        const onebit_hlayer_t &L = m.layers[i];
        hist |= L.dwa != nullptr;
        if (L.form == ONEBIT_LAYER_SEQUENTIAL) {
            const onebit_hff_t &f = L.ff;
            rm |= f.experts > 0;
            af = std::max<int64_t>(af, R * 16 * f.nt_plain);
            af = std::max<int64_t>(af, R * 8 * f.nt_gated);
            aux = std::max<int64_t>(aux, 16LL * f.nt_aux);
            if (f.experts) {
                const int64_t S = rup(expert_rows(f, R), 256) + 256;
                P.ez_rows = std::max<int64_t>({P.ez_rows, S, OB_EZ_ROWS});
                ae = std::max<int64_t>(ae, S * 8 * f.nt_expert);
                // tok_row, tok_w, gather | id_w | hist | blocks
                rt = std::max<int64_t>(rt, 2 * R * f.top + S + R + cdiv(R, OB_MOE_TOKENS) * f.experts + 4 * (std::min<int64_t>(f.experts, R * f.top) + R * f.top / 64 + 2));
            }
            as = std::max<int64_t>(as, R * 16 * L.side.nt);
        }
        if (L.kind == ONEBIT_MIX_LATENT_ATTENTION) {
            const onebit_hlatent_t &l = L.latent;
            const int64_t ra = rup(absorbed_rows(l, R, max_dec), 64);
            zc = std::max<int64_t>(zc, 16LL * L.nt_in);
            cq = std::max<int64_t>(cq, R * rup(l.q_rank, kt));
            qu = std::max<int64_t>(qu, R * L.heads * L.kp);
            qa = std::max<int64_t>(qa, ra * rup(L.heads, 16) * l.rp);
            lp = std::max<int64_t>(lp, (int64_t)OB_LAT_PARTS * L.heads * l.rp);
            lml = std::max<int64_t>(lml, 2LL * OB_LAT_PARTS * L.heads);
            if (l.flash) kv = std::max<int64_t>(kv, 2LL * L.heads * P.kv_rows * L.kp);
            am = std::max<int64_t>(am, R * L.mix_k);
            continue;
        }
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
    P.z = take((size_t)std::max<int64_t>(R, OB_ZROWS) * zc * 4);
    P.hist = take(hist ? (size_t)(m.n_runs + 1) * R * m.width * 4 : 0);
    P.hrm = take(rm ? (size_t)R * m.width_pad * es : 0);
    P.cq = take(cq * es);
    P.qu = take(qu * es);
    P.qa = take(qa * es);
    P.ctx = take(qa * es);
    P.lml = take(lml * 4);
    P.kv = take(kv * es);
    P.actm = take(am * es);
    P.actf = take(af * es);
    P.acte = take(ae * es);
    P.acts = take(as * es);
    P.spre = take((size_t)OB_SIDE_SPLITS * as * 4);
    P.ez = take((size_t)P.ez_rows * (P.ez_rows ? rup(m.width, 16) : 0) * 4);
    P.route = take(rt * 4);
    P.qn = take((size_t)R * qn * es);
    P.xbc = take((size_t)R * xbc * es);
    P.y = take((size_t)R * y * es);
    P.part = take(std::max<size_t>(max_splits > 1 ? (size_t)max_dec * max_splits * hd * 4 : 0, lp * 2));
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
        const bool att = L.kind == ONEBIT_MIX_SIGMOID_ATTENTION, seq = L.form == ONEBIT_LAYER_SEQUENTIAL;
        if (!att && L.kind != ONEBIT_MIX_SSM && L.kind != ONEBIT_MIX_LATENT_ATTENTION) return hfail(ONEBIT_E_ARG, "hybrid: layer %d: mixer kind %d", i, L.kind);
        if (!seq && L.form != ONEBIT_LAYER_PARALLEL) return hfail(ONEBIT_E_ARG, "hybrid: layer %d: form %d", i, L.form);
        if (seq) {
            const onebit_hff_t &f = L.ff;
            if (L.act_k || (L.kind != ONEBIT_MIX_LATENT_ATTENTION && L.nt_in != L.nt_mix + L.nt_aux)) return hfail(ONEBIT_E_SHAPE, "hybrid: layer %d: sequential layer with a merged feed-forward", i);
            if (f.nt_plain < 0 || (f.nt_plain & 1) || f.nt_gated < 0 || (f.nt_gated & 3) || f.nt_aux < 0 || (f.nt_aux & 1) || f.experts < 0 || (f.nt_plain && (f.nt_gated || f.nt_aux)) ||
                (f.nt_plain && (!f.w_plain_in || !f.w_plain_out)) || (f.nt_gated && (!f.w_gated_in || !f.w_gated_out)) || (f.nt_aux && !f.w_gated_in))
                return hfail(ONEBIT_E_SHAPE, "hybrid: layer %d: feed-forward sizes", i);
            if (!f.experts != !f.nt_aux) return hfail(ONEBIT_E_SHAPE, "hybrid: layer %d: experts without a router", i);
            if (f.experts) {
                const int n = f.experts + f.identity;
                if (f.identity < 0 || f.nt_expert <= 0 || (f.nt_expert & 3) || f.top <= 0 || f.groups <= 0 || n % f.groups || f.keep <= 0 || f.keep > f.groups ||
                    (int64_t)f.keep * (n / f.groups) < f.top || 16 * f.nt_aux < n || !f.w_expert_in || !f.w_expert_out || !f.correction)
                    return hfail(ONEBIT_E_SHAPE, "hybrid: layer %d: router sizes", i);
                ObRouteArgs ra = {};
                ra.experts = f.experts; ra.identity = f.identity; ra.groups = f.groups;
                ra.top = f.top;
                if (n > OB_MOE_MAX || ob_route_lds(ra) > 150 * 1024) return hfail(ONEBIT_E_SHAPE, "hybrid: layer %d: too many experts", i);
            }
            if (L.side.nt < 0 || (L.side.nt & 1) || (L.side.nt && (!L.side.w_gate || !L.side.w_proj || !L.side.norm_w || !L.side.table || L.side.dim <= 0 ||
                                                                    L.side.dim > 16 * L.side.nt || m->side_cols < L.side.dim)))
                return hfail(ONEBIT_E_SHAPE, "hybrid: layer %d: token input sizes", i);
        } else if (!L.norm_w || L.post1_w || L.pre2_w || L.post2_w || L.ff.nt_plain || L.ff.nt_gated || L.ff.experts || L.side.nt)
            return hfail(ONEBIT_E_ARG, "hybrid: layer %d: parallel layer with parts of a sequential one", i);
        if (L.kind == ONEBIT_MIX_LATENT_ATTENTION) {
            const onebit_hlatent_t &l = L.latent;
            const int64_t H = L.heads;
            if (!seq) return hfail(ONEBIT_E_ARG, "hybrid: layer %d: latent attention needs a sequential layer", i);
            if (!L.w_in || !L.w_out || !l.w_uq || !l.w_uk || !l.w_uv || !l.qn_w || !l.kvn_w || (l.flash && !l.w_kv)) return hfail(ONEBIT_E_ARG, "hybrid: layer %d: null pointer", i);
            if (H <= 0 || L.dim <= 0 || L.vdim <= 0 || l.q_rank <= 0 || l.kv_rank <= 0 || l.rp < l.kv_rank || l.rp % 32 || L.kp < L.dim || L.kp % 32 || l.vdp < L.vdim || l.vdp % 32 ||
                l.nt_q * 16 < l.q_rank || (L.nt_in - l.nt_q) * 16 < l.kv_rank || L.mix_k < H * l.vdp || L.mix_k % kt || L.b_in || L.b_out || l.q_rank + l.kv_rank > 32768 ||
                l.rp > 16384 || H * std::max(l.rp, L.kp) > 0x3fffffff)
                return hfail(ONEBIT_E_SHAPE, "hybrid: layer %d: latent attention sizes", i);
            if (l.tiled && (m->dtype != ONEBIT_HYB_BF16 || (l.rp != 64 && l.rp != 128 && l.rp != 256 && l.rp != 512))) return hfail(ONEBIT_E_SHAPE, "hybrid: layer %d: tiled latent attention sizes", i);
            if (l.flash && (!l.tiled || (L.kp != 64 && L.kp != 128) || l.vdp > L.kp || (int64_t)m->max_len * L.kp * 2 > 0x7fffffffLL)) return hfail(ONEBIT_E_SHAPE, "hybrid: layer %d: expanded latent attention sizes", i);
            continue;
        }
        if (!L.w_in || !L.w_out || (!seq && !L.norm_w) || L.heads <= 0 || L.vdim <= 0 || L.nt_mix <= 0 || L.nt_aux < 0 || ((L.nt_mix + L.nt_aux) & 1) ||
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
        if (m->runs[i].layer < 0 || m->runs[i].layer >= m->n_layers || !m->runs[i].s0 ||
            (!m->runs[i].s1 && m->layers[m->runs[i].layer].kind != ONEBIT_MIX_LATENT_ATTENTION)) return hfail(ONEBIT_E_ARG, "hybrid: run %d", i);
    if (m->bigram && (!m->token_history || m->buckets <= 0 || m->mul_prev < 0 || m->mul_cur < 0)) return hfail(ONEBIT_E_ARG, "hybrid: bigram table");
    return 0;
}

extern "C" size_t onebit_hybrid_workspace_bytes(const onebit_hmodel_t *m, int64_t max_rows, int64_t max_out, int32_t max_dec, int32_t max_splits)
{
    HPlan P;
    if (check_model(m) || max_rows <= 0 || max_dec < 0 || max_splits < 1 || make_plan(*m, max_rows, max_out, max_dec, max_splits, P)) return 0;
    return P.total;
}

// ---------------------------------------------------------------------------------------------------------------- step --
// the row kernel between two products; the wider form only where a layer needs it
template <typename E>
static int row_launch(const ObXRowArgs &a, int rows, hipStream_t s)
{
    if (rows <= 0) return 0;
    const bool ext = a.post_w || a.top || a.id_w || a.hist || a.out_rm || !a.w || (a.embed && (a.bigram || a.embed_scale != 1.0f));
    const int lds = (((a.W + 3) & ~3) + 16) * 4;
    const unsigned thr = (unsigned)std::min<int64_t>(rows <= 256 || ext ? 1024 : 512, std::max<int64_t>(64, rup(cdiv(a.W, 4), 64)));
    auto go = [&](auto kern, const auto &args) {
        if (!lds_ok((const void *)kern, lds)) return hfail(ONEBIT_E_SHAPE, "row kernel: LDS");
        hipLaunchKernelGGL(kern, dim3((unsigned)rows), dim3(thr), lds, s, args);
        return hstatus("row kernel");
    };
    if (ext) {
        const bool one = a.W <= 4 * (int)thr;
#define OB_XROW(K) (a.W % 4 == 0 ? one ? go(ob_xrow_kernel<E, 4, true, K>, a) : go(ob_xrow_kernel<E, 4, false, K>, a) : go(ob_xrow_kernel<E, 1, false, K>, a))
        return a.embed ? OB_XROW(OB_X_EMBED) : a.top && a.hist ? OB_XROW(OB_X_BOTH) : a.top ? OB_XROW(OB_X_EXPERTS) : a.hist ? OB_XROW(OB_X_DEPTH) : OB_XROW(OB_X_PLAIN);
#undef OB_XROW
    }
    const ObHNormArgs &n = a;
    return a.W % 4 == 0 ? go(ob_hnorm_kernel<E, 4>, n) : go(ob_hnorm_kernel<E, 1>, n);
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

// plain product into fp32 partial sums: returns the number of splits through n_split
template <typename E>
static int part_launch(ObDenseArgs d, float *z, int &n_split, hipStream_t s)
{
    d.z = z; d.ldz = 16 * d.n_tiles; d.z_split = (size_t)d.T * d.ldz;
    n_split = gemm_splits(d.n_tiles, d.nkt, d.T);
    n_split = (int)cdiv(d.nkt, cdiv(d.nkt, n_split));
    return dense_launch<E, OB_EPI_PART>(d, n_split, s);
}

// latent attention up to its heads' outputs, in `act` (the rows of the output product)
template <typename E>
static int latent_launch(const onebit_hmodel_t &m, const onebit_hlayer_t &L, const onebit_hrun_t &run, const onebit_hstate_t &st, const HPlan &P,
                         char *ws, void *act, int act_nkt, hipStream_t s)
{
    constexpr int KT = ObElem<E>::KT;
    const onebit_hlatent_t &l = L.latent;
    const int T = st.n_rows, H = L.heads, bands = (int)cdiv(m.max_len, 16), cq_nkt = (int)cdiv(l.q_rank, KT);
    float *z = (float *)(ws + P.z);
    int n_split;
    ObDenseArgs d = {};
    d.w = L.w_in; d.a = ws + P.h; d.n_tiles = L.nt_in; d.nkt = m.width_pad / KT; d.T = T;
    if (int rc = part_launch<E>(d, z, n_split, s)) return rc;
    ObLatPrepArgs p = {z, (size_t)T * 16 * L.nt_in, n_split, 16 * L.nt_in, l.q_rank, 16 * l.nt_q, l.kv_rank, l.qn_w, l.kvn_w, m.eps, ws + P.cq, cq_nkt, run.s0, l.rp, bands,
                       st.row_slot, st.row_pos, m.n_slots, m.max_len};
    const int n_in = l.q_rank + l.kv_rank, plds = (((n_in + 3) & ~3) + 16) * 4;
    const bool vec = l.q_rank % 4 == 0 && l.kv_rank % 4 == 0;
    auto pgo = [&](auto pk) {
        if (!lds_ok((const void *)pk, plds)) return hfail(ONEBIT_E_SHAPE, "latent norms: LDS");
        hipLaunchKernelGGL(pk, dim3((unsigned)T), dim3((unsigned)std::min<int64_t>(T <= 256 ? 1024 : 512, rup(cdiv(n_in, vec ? 4 : 1), 64))), plds, s, p);
        return hstatus("latent norms");
    };
    if (int rc = vec ? pgo(ob_lat_prep_kernel<E, 4>) : pgo(ob_lat_prep_kernel<E, 1>)) return rc;
    // queries, row-major [T][H kp]
    ObDenseArgs q = {};
    q.w = l.w_uq; q.a = ws + P.cq; q.n_tiles = q.nt_mix = H * L.kp / 16; q.nkt = cq_nkt; q.T = T; q.u = ws + P.qu;
    if (int rc = dense_launch<E, OB_EPI_IN>(q, 1, s)) return rc;
    int n_abs = T;
    int first = st.n_seg;
    if (l.tiled && l.flash) {
        n_abs = st.n_dec;
        for (first = 0; first < st.n_short; ++first) n_abs += st.segs[first].n;
    }
    if (n_abs) {
        ObDenseArgs k = {};
        k.w = l.w_uk; k.a = ws + P.qu; k.lda = H * L.kp; k.tile_group = l.rp / 16; k.act_cols = L.kp; k.n_tiles = k.nt_mix = H * l.rp / 16; k.nkt = L.kp / KT; k.T = n_abs; k.u = ws + P.qa;
        if constexpr (sizeof(E) == 2) {
            if (l.tiled) {
                k.heads = ws + P.qa; k.head_rows = (int)cdiv(H, 16);
                for (k.d_shift = 6; (1 << k.d_shift) < l.rp; ++k.d_shift) {}
                if (int rc = dense_heads_launch<E, OB_EPI_QFRAG>(k, (size_t)OB_SKINNY_T * rup(H, 16) * l.rp * sizeof(E), s)) return rc;
            }
        }
        if (!l.tiled) if (int rc = dense_heads_launch<E, OB_EPI_IN>(k, (size_t)OB_SKINNY_T * H * l.rp * sizeof(E), s)) return rc;
        ObLatArgs a = {ws + P.qa, ws + P.ctx, H * l.rp, run.s0, l.rp, bands, st.row_slot, st.row_pos, 0, H, m.n_slots, m.max_len, L.scale, 0, 1, ws + P.part, (float *)(ws + P.lml)};
        if (!l.tiled) {
            auto rk = ob_lat_rows_kernel<E>;
            const int lds = (l.rp + 256 + 16) * 4;
            if (!lds_ok((const void *)rk, lds)) return hfail(ONEBIT_E_SHAPE, "latent attention: LDS");
            for (int r0 = 0; r0 < n_abs; r0 += 32768) {
                a.row0 = r0;
                hipLaunchKernelGGL(rk, dim3((unsigned)H, (unsigned)std::min(n_abs - r0, 32768)), dim3(256), lds, s, a);
            }
        } else {
            int ctx = 1;                                              // longest context of the absorbed rows
            if (st.n_dec || st.n_short) ctx = st.attn_chunk * st.attn_splits;
            for (int i = st.n_short; i < (first == st.n_seg ? st.n_seg : 0); ++i) ctx = std::max(ctx, st.segs[i].past + st.segs[i].n);
            const int ht = H > 16 && l.rp <= 512 ? 2 : 1, hg = (int)cdiv(H, 16 * ht);
            // as many workgroups as run at once (their LDS decides: one per CU at 512 columns); every split writes all heads' outputs for the
            // combining launch to read, so never more than that, and at most 32
            const int per_cu = l.rp >= 512 ? 1 : l.rp >= 256 ? 2 : 4;
            const int64_t want = std::min<int64_t>({256 * per_cu / ((int64_t)n_abs * hg), cdiv(ctx, 64), OB_LAT_PARTS / n_abs, 32});
            a.chunk = (int)rup(cdiv(ctx, std::max<int64_t>(1, want)), 64);
            a.nsplit = (int)cdiv(ctx, a.chunk);
            for (int r0 = 0; r0 < n_abs; r0 += 32768) {
                a.row0 = r0;
                const dim3 grid((unsigned)hg, (unsigned)std::min(n_abs - r0, 32768), (unsigned)a.nsplit);
                auto go = [&](auto kern, int rp) {
                    const int lds = 2 * rp * 128 + 16 * ht * 68 * 4;
                    if (!lds_ok((const void *)kern, lds)) return hfail(ONEBIT_E_SHAPE, "latent attention: LDS");
                    hipLaunchKernelGGL(kern, grid, dim3(256 * ht), lds, s, a);
                    return hstatus("latent attention");
                };
                int rc;
                if constexpr (sizeof(E) == 2) {
                    if (ht == 2) rc = l.rp == 64 ? go(ob_lat_dec_kernel<64, 2>, 64) : l.rp == 128 ? go(ob_lat_dec_kernel<128, 2>, 128)
                                    : l.rp == 256 ? go(ob_lat_dec_kernel<256, 2>, 256) : go(ob_lat_dec_kernel<512, 2>, 512);
                    else rc = l.rp == 64 ? go(ob_lat_dec_kernel<64, 1>, 64) : l.rp == 128 ? go(ob_lat_dec_kernel<128, 1>, 128)
                            : l.rp == 256 ? go(ob_lat_dec_kernel<256, 1>, 256) : go(ob_lat_dec_kernel<512, 1>, 512);
                } else rc = hfail(ONEBIT_E_DTYPE, "latent attention: tiled form in fp32");
                if (rc) return rc;
                if (a.nsplit > 1) hipLaunchKernelGGL(ob_lat_combine_kernel, dim3((unsigned)H, grid.y), dim3((unsigned)std::min<int64_t>(256, rup(l.rp / 8, 64))), 0, s, a);
            }
        }
        if (int rc = hstatus("latent attention")) return rc;
        ObDenseArgs v = {};
        v.w = l.w_uv; v.a = ws + P.ctx; v.lda = H * l.rp; v.tile_group = l.vdp / 16; v.act_cols = l.rp; v.n_tiles = H * l.vdp / 16; v.nkt = l.rp / KT; v.T = n_abs;
        v.act = act; v.act_nkt = act_nkt; v.fn = OB_FN_ID;
        if (int rc = dense_heads_launch<E, OB_EPI_ACT>(v, (size_t)(OB_SKINNY_T / 16) * act_nkt * 1024, s)) return rc;
    }
    if constexpr (sizeof(E) == 2) {
        // prompts: the keys and values of as many chunks as the buffer holds, then their attention
        const int sh = L.kp == 64 ? 6 : 7;
        for (int s0 = first; s0 < st.n_seg;) {
            ObDenseSegArgs e = {};
            ObFlashSigArgs f = {};
            int64_t rows = 0, wgs = 0;
            int64_t keys = 0;
            for (int i = s0; i < st.n_seg && e.nseg < OB_DENSE_MAXSEG; ++i) keys += st.segs[i].past + st.segs[i].n;
            const bool big = cdiv(2 * H * L.kp, 256) * cdiv(std::min(keys, P.kv_rows), 256) >= 224;
            const int br = big ? 256 : 128;
            int blocks = 0, i = s0;
            for (; i < st.n_seg && e.nseg < OB_DENSE_MAXSEG; ++i) {
                const onebit_hseg_t &g = st.segs[i];
                const int len = g.past + g.n, n = e.nseg;
                if (rows + rup(len, 16) > P.kv_rows) break;
                blocks += (int)cdiv(len, br);
                e.blk_end[n] = blocks; e.band0[n] = g.slot * bands; e.row0[n] = (int)rows; e.rows[n] = len;
                wgs += (cdiv(g.n, OB_FL_BM) + 1) / 2 * H;
                if (wgs > 0x3fffffffLL) return hfail(ONEBIT_E_ARG, "attention: too many workgroups");
                f.wg_end[n] = (int)wgs;
                f.seg[n] = {g.row0, g.n, (int)rows, g.past};
                f.nseg = ++e.nseg;
                rows += rup(len, 16);
            }
            if (i == s0) return hfail(ONEBIT_E_SHAPE, "latent attention: chunk %d does not fit the expansion buffer", s0);
            e.w = l.w_kv; e.a = run.s0; e.n_tiles = 2 * H * L.kp / 16; e.nkt = l.rp / KT; e.kt_split = e.nkt; e.T = blocks * br;
            e.heads = ws + P.kv; e.d_shift = sh; e.head_rows = (int)P.kv_rows;
            auto go = [&](auto kern, int nb, int thr, int lds) {
                if (!lds_ok((const void *)kern, lds)) return hfail(ONEBIT_E_SHAPE, "expansion: LDS");
                hipLaunchKernelGGL(kern, dim3((unsigned)(cdiv(e.n_tiles, nb) * blocks)), dim3(thr), lds, s, e);
                return hstatus("expansion");
            };
            const int rc = big ? go(ob_dense_tile_kernel<E, OB_EPI_HEADS, 16, 16, 2, 4, 4, OB_ROWS_SEGS>, 16, 512, 128 * 1024)
                               : go(ob_dense_tile_kernel<E, OB_EPI_HEADS, 8, 8, 2, 2, 4, OB_ROWS_SEGS>, 8, 256, 64 * 1024);
            if (rc) return rc;
            f.a.q = (const _Float16 *)(ws + P.qu); f.a.k = (const _Float16 *)(ws + P.kv); f.a.v = f.a.k + (size_t)H * P.kv_rows * L.kp;     // (bf16 behind these pointers)
            f.a.H = f.a.Hkv = H; f.a.max_len = (int)P.kv_rows;
            f.a.scale_log2e = L.scale * OB_LOG2E;
            f.out = act; f.out_nkt = act_nkt; f.vdim = l.vdp;
            if (L.kp == 128) hipLaunchKernelGGL((ob_flash_fwd_kernel<128, true, ObFlSoftmaxBf16>), dim3((unsigned)wgs), dim3(256), 0, s, f);
            else hipLaunchKernelGGL((ob_flash_fwd_kernel<64, true, ObFlSoftmaxBf16>), dim3((unsigned)wgs), dim3(256), 0, s, f);
            if (int rc2 = hstatus("prompt attention")) return rc2;
            s0 = i;
        }
    }
    return 0;
}

// the feed-forward of a sequential layer; what the next row kernel adds goes into `pend`
template <typename E>
static int ff_launch(const onebit_hmodel_t &m, const onebit_hlayer_t &L, const onebit_hstate_t &st, const HPlan &P, char *ws, ObXRowArgs &pend, hipStream_t s)
{
    constexpr int KT = ObElem<E>::KT;
    const onebit_hff_t &f = L.ff;
    const int T = st.n_rows, w_nkt = m.width_pad / KT, wt = (int)cdiv(m.width, 16);
    auto out_product = [&](const void *w, int nkt) -> int {
        ObDenseArgs o = {};
        o.w = w; o.a = ws + P.actf; o.n_tiles = wt; o.nkt = nkt; o.T = T;
        pend.z = (float *)(ws + P.z); pend.ldz = 16 * wt; pend.z_split = (size_t)T * pend.ldz;
        return part_launch<E>(o, (float *)(ws + P.z), pend.n_split, s);
    };
    ObDenseArgs d = {};
    d.a = ws + P.h; d.nkt = w_nkt; d.T = T; d.act = ws + P.actf;
    if (f.nt_plain) {
        d.w = f.w_plain_in; d.n_tiles = f.nt_plain; d.act_nkt = 16 * f.nt_plain / KT; d.fn = OB_FN_XIELU; d.fa = f.act_a; d.fb = f.act_b;
        if (int rc = dense_launch<E, OB_EPI_ACT>(d, 1, s)) return rc;
        return out_product(f.w_plain_out, d.act_nkt);
    }
    if (f.nt_gated + f.nt_aux) {
        d.w = f.w_gated_in; d.n_tiles = f.nt_aux + f.nt_gated; d.aux = (float *)(ws + P.aux); d.nt_aux = f.nt_aux; d.act_nkt = 8 * f.nt_gated / KT;
        if (int rc = dense_launch<E, OB_EPI_IN>(d, 1, s)) return rc;
        if (f.nt_gated) if (int rc = out_product(f.w_gated_out, d.act_nkt)) return rc;
    }
    if (!f.experts) return 0;
    const int64_t TK = (int64_t)T * f.top, S = expert_rows(f, T);
    if ((int64_t)T * m.width_pad * (int)sizeof(E) > 0xffffffffLL || S > 0x7fffffff / 16) return hfail(ONEBIT_E_SHAPE, "experts: %d rows in one step", T);
    const int64_t live = std::min<int64_t>(f.experts, TK);
    int br = OB_SKINNY_T;
    if (T > OB_SKINNY_T) br = sizeof(E) == 2 && TK / f.experts >= 384 ? 256 : 128;
    const int n_blk = (int)(live + (br == OB_SKINNY_T ? 0 : TK / br));
    ObRouteArgs r = {};
    int32_t *at = (int32_t *)(ws + P.route);
    r.z = (const float *)(ws + P.aux); r.ldz = 16 * f.nt_aux; r.correction = f.correction;
    r.T = T; r.experts = f.experts; r.identity = f.identity; r.top = f.top; r.groups = f.groups; r.keep = f.keep;
    const int n_wg = (int)cdiv(T, OB_MOE_TOKENS);
    r.blk = (ObRowBlock *)at; at += 4 * n_blk;
    r.tok_row = at; at += TK;
    r.tok_w = (float *)at; at += TK;
    r.id_w = (float *)at; at += T;
    r.gather = at; at += S;
    r.hist = at;
    r.block_rows = br; r.n_blk = n_blk;
    const int lds = (int)ob_route_lds(r), n_all = f.experts + f.identity;
    auto route = [&](auto k) {
        if (!lds_ok((const void *)k, lds)) return hfail(ONEBIT_E_SHAPE, "router: LDS");
        hipLaunchKernelGGL(k, dim3((unsigned)n_wg), dim3(1024), lds, s, r);
        return 0;
    };
#define OB_ROUTE(S) (n_all <= 64 ? route(ob_route_kernel<S, 1>) : n_all <= 256 ? route(ob_route_kernel<S, 4>) : route(ob_route_kernel<S, 16>))
    if (int rc = n_wg == 1 ? OB_ROUTE(true) : OB_ROUTE(false)) return rc;
#undef OB_ROUTE
    if (n_wg > 1) {
        const int runs = std::max(1, 1024 / f.experts);
        hipLaunchKernelGGL(ob_route_scan_kernel, dim3(1), dim3(1024), f.experts * 4 * (runs + 1), s, r, n_wg, runs);
        hipLaunchKernelGGL(ob_route_rows_kernel, dim3((unsigned)n_wg), dim3(256), f.experts * 4, s, r);
    }
    if (int rc = hstatus("router")) return rc;
    ObDenseArgs u = {};
    u.w = f.w_expert_in; u.a = ws + P.hrm; u.lda = m.width_pad; u.n_tiles = f.nt_expert; u.nkt = w_nkt; u.T = T; u.w_group = (size_t)f.nt_expert * w_nkt;
    u.act = ws + P.acte; u.act_nkt = 8 * f.nt_expert / KT; u.blk = r.blk; u.gather = r.gather;
    if (int rc = dense_blocks_launch<E, OB_EPI_IN, OB_ROWS_GATHER>(u, n_blk, br, 1, s)) return rc;
    ObDenseArgs o = {};
    o.w = f.w_expert_out; o.a = ws + P.acte; o.n_tiles = wt; o.nkt = u.act_nkt; o.T = T; o.w_group = (size_t)wt * o.nkt;
    o.z = (float *)(ws + P.ez); o.ldz = 16 * wt; o.z_split = (size_t)S * o.ldz; o.blk = r.blk;
    int n_split = 1;
    if (br == OB_SKINNY_T) n_split = (int)std::max<int64_t>(1, std::min<int64_t>({cdiv(512, cdiv(wt, 2) * live), o.nkt / 8, OB_EZ_ROWS / S, 8}));
    n_split = (int)cdiv(o.nkt, cdiv(o.nkt, n_split));
    if (br == OB_SKINNY_T) {
        if (int rc = dense_blocks_launch<E, OB_EPI_PART, OB_ROWS_SORTED>(o, n_blk, br, n_split, s)) return rc;
        pend.ez = o.z;
    } else {                                                          // many rows: outputs in the work type, half the traffic
        o.u = o.z; o.nt_mix = wt;
        if (int rc = dense_blocks_launch<E, OB_EPI_IN, OB_ROWS_SORTED>(o, n_blk, br, 1, s)) return rc;
        pend.eo = o.u;
    }
    pend.ez_split = o.z_split; pend.ez_n = n_split; pend.ld_ez = o.ldz; pend.top = f.top; pend.tok_row = r.tok_row; pend.tok_w = r.tok_w;
    if (f.identity) {
        pend.id_w = r.id_w;
        if (L.pre2_w) { pend.idh = ws + P.hrm; pend.ld_idh = m.width_pad; }
    }
    return 0;
}

// the token's own input: gate product, gelu and the token's row, output product
template <typename E>
static int side_launch(const onebit_hmodel_t &m, const onebit_hlayer_t &L, const onebit_hstate_t &st, const HPlan &P, char *ws, int &n_split, hipStream_t s)
{
    constexpr int KT = ObElem<E>::KT;
    const int T = st.n_rows, nkt = 16 * L.side.nt / KT;
    ObDenseArgs g = {}, o = {};
    g.w = L.side.w_gate; g.a = ws + P.h; g.n_tiles = L.side.nt; g.nkt = m.width_pad / KT; g.T = T;
    o.w = L.side.w_proj; o.n_tiles = (int)cdiv(m.width, 16); o.nkt = nkt; o.T = T;
    o.table = L.side.table; o.ld_table = m.side_cols; o.table_cols = L.side.dim; o.tokens = st.tokens;
    float *pre = (float *)(ws + P.spre);
    g.z = pre; g.ldz = 16 * L.side.nt; g.z_split = (size_t)T * g.ldz;
    const int64_t wgs = T <= OB_SKINNY_T ? cdiv(g.n_tiles, 2) : cdiv(g.n_tiles, 8) * cdiv(T, 128);
    int n_pre = (int)std::max<int64_t>(1, std::min<int64_t>({cdiv(512, wgs), g.nkt / 16, OB_SIDE_SPLITS}));
    n_pre = (int)cdiv(g.nkt, cdiv(g.nkt, n_pre));
    if (int rc = dense_launch<E, OB_EPI_PART>(g, n_pre, s)) return rc;
    o.pre = pre; o.n_pre = n_pre; o.ld_pre = g.ldz;
    const int mt = T <= 16 ? 1 : T <= 32 ? 2 : 4, lds = mt * nkt * 1024;
    if (T <= OB_SKINNY_T && lds <= 48 * 1024) {                       // few rows: the output product forms its own operand
        o.z = (float *)(ws + P.z); o.ldz = 16 * o.n_tiles; o.z_split = (size_t)T * o.ldz; o.kt_split = o.nkt;
        n_split = 1;
        const dim3 grid((unsigned)cdiv(o.n_tiles, 2));
        if (mt == 1) hipLaunchKernelGGL((ob_dense_skinny_kernel<E, OB_EPI_PART, 1, OB_ROWS_TABLE>), grid, dim3(256), lds, s, o);
        else if (mt == 2) hipLaunchKernelGGL((ob_dense_skinny_kernel<E, OB_EPI_PART, 2, OB_ROWS_TABLE>), grid, dim3(256), lds, s, o);
        else hipLaunchKernelGGL((ob_dense_skinny_kernel<E, OB_EPI_PART, 4, OB_ROWS_TABLE>), grid, dim3(256), lds, s, o);
        return hstatus("token input");
    }
    o.act = ws + P.acts;
    hipLaunchKernelGGL(ob_table_rows_kernel<E>, dim3((unsigned)cdiv((int64_t)T * nkt * KT / 4, 256)), dim3(256), 0, s, o);
    if (int rc = hstatus("token input")) return rc;
    o.a = o.act;
    return part_launch<E>(o, (float *)(ws + P.z), n_split, s);
}

template <typename E>
static int step_impl(const onebit_hmodel_t &m, const onebit_hstate_t &st, const HPlan &P, hipStream_t s)
{
    constexpr int KT = ObElem<E>::KT;
    char *ws = (char *)st.workspace;
    const int T = st.n_rows, ldz = (int)rup(m.width, 16), w_nkt = m.width_pad / KT;
    bool loop = false, hist = false;
    for (int i = 0; i < m.n_runs; ++i) { loop |= m.runs[i].add_embedding != 0; hist |= m.layers[m.runs[i].layer].dwa != nullptr; }
    ObXRowArgs nb = {};
    nb.x = (float *)(ws + P.x); nb.ldz = ldz; nb.mult = m.mult; nb.off = m.norm_off; nb.eps = m.eps; nb.W = m.width; nb.out_nkt = w_nkt;
    nb.tokens = st.tokens; nb.row_pos = st.row_pos; nb.row_slot = st.row_slot; nb.row_off = st.row_off; nb.n_slots = m.n_slots; nb.max_len = m.max_len;
    nb.embed_scale = m.embed_scale; nb.ld_rm = m.width_pad;
    // what the next row kernel adds to the residual: nothing yet (the embedding), or the last sublayer's output
    ObXRowArgs pend = nb;
    pend.embed = m.embed; pend.pos_embed = m.pos_embed; pend.bigram = m.bigram; pend.buckets = m.buckets; pend.mul_prev = m.mul_prev; pend.mul_cur = m.mul_cur;
    pend.tok_hist = m.token_history;
    if (loop) pend.emb_save = (float *)(ws + P.emb0);
    auto keep_result = [&](int i, const float *dwa) {                 // X_i
        if (!hist) return;
        pend.hist = (float *)(ws + P.hist); pend.hist_stride = (size_t)T * m.width; pend.hist_i = i; pend.dwa = dwa;
    };
    keep_result(0, nullptr);
    auto residual_out = [&](int run) -> int {      // x + (pending product), without touching the stream's own copy
        if (!st.residuals) return 0;
        float *dst = st.residuals + (size_t)run * T * m.width;
        const hipError_t e = hipMemcpyAsync(dst, ws + P.x, (size_t)T * m.width * 4, hipMemcpyDeviceToDevice, s);
        if (e != hipSuccess) return hfail((int)e, "residual copy: %s", hipGetErrorString(e));
        ObXRowArgs a = pend;
        a.x = dst; a.w = m.final_norm; a.out = ws + P.out_h;      // (norm output unused; see the size check in onebit_hybrid_step)
        a.emb_save = nullptr;
        return row_launch<E>(a, T, s);
    };
    for (int r = 0; r < m.n_runs; ++r) {
        const onebit_hrun_t &run = m.runs[r];
        const onebit_hlayer_t &L = m.layers[run.layer];
        const bool latent = L.kind == ONEBIT_MIX_LATENT_ATTENTION;
        const int act_nkt = (L.mix_k + L.act_k) / KT;
        void *act = ws + (latent ? P.actm : P.act[act_index(P, L)]);
        ObXRowArgs a = pend;
        a.w = L.norm_w; a.out = ws + P.h;
        if (run.add_embedding) a.emb_add = (const float *)(ws + P.emb0);
        if (int rc = row_launch<E>(a, T, s)) return rc;
        if (latent) {
            if (int rc = latent_launch<E>(m, L, run, st, P, ws, act, act_nkt, s)) return rc;
        } else {
            ObDenseArgs d = {};
            d.w = L.w_in; d.a = ws + P.h; d.n_tiles = L.nt_in; d.nkt = w_nkt; d.T = T;
            d.bias = L.b_in; d.u = ws + P.u; d.nt_mix = L.nt_mix; d.aux = (float *)(ws + P.aux); d.nt_aux = L.nt_aux;
            d.act = act; d.act_k0 = L.mix_k; d.act_nkt = act_nkt;
            if (int rc = dense_launch<E, OB_EPI_IN>(d, 1, s)) return rc;
            const int rc = L.kind == ONEBIT_MIX_SIGMOID_ATTENTION ? attention_launch<E>(m, L, run, st, P, ws, act, act_nkt, s)
                                                                  : ssm_launch<E>(m, L, run, st, P, ws, act, act_nkt, s);
            if (rc) return rc;
        }
        ObDenseArgs o = {};
        o.w = L.w_out; o.a = act; o.n_tiles = ldz / 16; o.nkt = act_nkt; o.T = T;
        pend = nb;
        pend.z = (float *)(ws + P.z); pend.z_split = (size_t)T * ldz; pend.bias = L.b_out; pend.post_w = L.post1_w;
        if (int rc = part_launch<E>(o, (float *)(ws + P.z), pend.n_split, s)) return rc;
        if (L.form == ONEBIT_LAYER_SEQUENTIAL) {
            const onebit_hff_t &f = L.ff;
            if (f.nt_plain || f.nt_gated || f.experts) {
                a = pend;
                a.w = L.pre2_w; a.out = ws + P.h;
                if (f.experts) a.out_rm = ws + P.hrm;
                if (int rc = row_launch<E>(a, T, s)) return rc;
                pend = nb;
                pend.post_w = L.post2_w;
                if (int rc = ff_launch<E>(m, L, st, P, ws, pend, s)) return rc;
            }
            if (L.side.nt) {
                a = pend;
                a.w = nullptr; a.out = ws + P.h;
                if (int rc = row_launch<E>(a, T, s)) return rc;
                pend = nb;
                pend.mult = 1.0f;
                pend.z = (float *)(ws + P.z); pend.z_split = (size_t)T * ldz; pend.post_w = L.side.norm_w;
                if (int rc = side_launch<E>(m, L, st, P, ws, pend.n_split, s)) return rc;
            }
        }
        keep_result(r + 1, L.dwa);
        if (int rc2 = residual_out(r)) return rc2;
    }
    if (st.n_out > 0) {
        ObXRowArgs a = pend;
        a.w = m.final_norm; a.out = ws + P.out_h; a.rows = st.out_rows; a.emb_save = nullptr;
        if (int rc = row_launch<E>(a, st.n_out, s)) return rc;
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
    if (st->n_short < 0 || st->n_short > st->n_seg) return hfail(ONEBIT_E_ARG, "hybrid_step: n_short %d of %d chunks", st->n_short, st->n_seg);
    if ((st->n_dec || st->n_short) && (st->attn_splits < 1 || st->attn_chunk < 128 || st->attn_chunk % 128)) return hfail(ONEBIT_E_SHAPE, "hybrid_step: attn_chunk must be a multiple of 128");
    if (st->residuals && st->n_rows > rup(std::max<int64_t>(max_out, 1), 256)) return hfail(ONEBIT_E_SHAPE, "hybrid_step: residuals need room for n_rows output rows");
    int row = st->n_dec;
    for (int i = 0; i < st->n_seg; ++i) {
        const onebit_hseg_t &g = st->segs[i];
        if (g.row0 != row || g.n < 1 || g.slot < 0 || g.slot >= m->n_slots || g.past < 0 || (int64_t)g.past + g.n > m->max_len)
            return hfail(ONEBIT_E_SHAPE, "hybrid_step: segment %d (rows %d + %d, slot %d, past %d)", i, g.row0, g.n, g.slot, g.past);
        if (i < st->n_short && (g.n > ONEBIT_HYB_SHORT || st->n_dec + st->n_seg > max_dec || (int64_t)g.past + g.n > (int64_t)st->attn_chunk * st->attn_splits))
            return hfail(ONEBIT_E_SHAPE, "hybrid_step: chunk %d is not a short one", i);
        row += g.n;
    }
    if (row != st->n_rows) return hfail(ONEBIT_E_SHAPE, "hybrid_step: n_rows %d, decode rows and segments make %d", st->n_rows, row);
    HPlan P;
    if (int rc = make_plan(*m, max_rows, max_out, max_dec, max_splits, P)) return rc;
    if (st->workspace_bytes < P.total || ((uintptr_t)st->workspace & 255)) return hfail(ONEBIT_E_WSPACE, "hybrid_step: workspace %zu of %zu bytes (256-byte aligned)", st->workspace_bytes, P.total);
    return m->dtype == ONEBIT_HYB_BF16 ? step_impl<__bf16>(*m, *st, P, (hipStream_t)stream) : step_impl<float>(*m, *st, P, (hipStream_t)stream);
}
