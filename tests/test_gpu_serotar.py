"""Serotar on the GPU against the plain restatement (oracle/serotar_ref.py, float64): each mechanism alone, prompts, decoding through the cache,
portions, batches, slots used again, far keys, odd sizes, generation through the scheduler.

Weights are random bf16, so the restatement runs on the very numbers the kernels read; what remains is the rounding of bf16 activations
(``TOL``), or fp32 rounding.  A choice between experts that is decided by less than that rounding may fall differently: bf16 comparisons leave
out the positions where the restatement finds such a choice (``clear``)."""
import json

import pytest
import torch

from onebit_amd.serotar import SerotarConfig, SerotarForCausalLM, synthetic_weights
from oracle import lebepel_ref, serotar_ref as R
from test_serotar_cpu import dense, layer, moe, raw_config

pytestmark = pytest.mark.gpu
BF, F32 = torch.bfloat16, torch.float32
TOL = {BF: 0.03, F32: 3e-5}
DTYPES = pytest.mark.parametrize("dtype", [BF, F32], ids=["bf16", "f32"])


def build(raw, dtype, seed=0, edit=None):
    cfg = SerotarConfig.from_dict(raw)
    w = synthetic_weights(cfg, seed)
    if edit is not None:
        edit(w)
    return SerotarForCausalLM(cfg, w, dtype), w


def tokens(n, vocab, seed=0):
    return torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def rows_err(got, want):
    got, want = got.double().cpu(), want.double()
    return (got - want).pow(2).mean(-1).sqrt() / want.pow(2).mean().sqrt()


def err(got, want, ok=None):
    """The largest row error: rms of the difference over the rms of the whole reference."""
    e = rows_err(got, want)
    return float((e if ok is None else e[ok]).max())


def run(eng, slot, start, toks):
    eng.launch([(slot, start, toks, list(range(len(toks))))])
    return eng.logits[:len(toks)].clone()


def run_cut(eng, slot, toks, cuts):
    out, at = [], 0
    for n in cuts:
        out.append(run(eng, slot, at, toks[at:at + n]))
        at += n
    while at < len(toks):                                                      # the rest one by one (graph replays)
        eng.launch([(slot, at, toks[at:at + 1])])
        out.append(eng.logits[:1].clone())
        at += 1
    return torch.cat(out)


def clear_choices(raw, w, toks, gap=0.06):
    """Positions at which no layer's choice of experts (or of groups) is close: the last one in and the first one out differ by more than ``gap``
    of the larger score."""
    ok = torch.ones(len(toks), dtype=torch.bool)
    true_choose = R.choose

    def watch(s, correction, router):
        choice = (s + correction)
        n, g = len(choice), router.get("groups") or dict(count=1, keep=1)
        size = n // g["count"]
        m = choice.view(g["count"], size).max(-1).values.sort(descending=True).values
        margin = 1.0 if g["keep"] == g["count"] else float((m[g["keep"] - 1] - m[g["keep"]]) / m[g["keep"] - 1].abs())
        got = true_choose(s, correction, router)
        best = choice.view(g["count"], size).max(-1).values.argsort(descending=True)[:g["keep"]].tolist()
        left = [float(choice[i]) for i in range(n) if i // size in best and i not in got]
        if left:
            low = min(float(choice[i]) for i in got)
            margin = min(margin, (low - max(left)) / max(abs(low), 1e-9))
        seen.append(margin)
        return got
    seen = []
    R.choose = watch
    try:
        ref = R.forward(raw, w, toks)
    finally:
        R.choose = true_choose
    if seen:
        ok = torch.tensor(seen).view(-1, len(toks)).min(0).values > gap
    return ref, ok


def only(*keep):
    """An edit that silences the parts of layer 0 that are not named: output norms' weights to zero, the depth average to the last result."""
    def edit(w):
        for part, name in (("mix", "l0.ls1"), ("mlp", "l0.ls2"), ("side", "l0.side.norm")):
            if part not in keep and name in w:
                w[name].zero_()
        w["l0.dwa"].copy_(torch.tensor([0.0, 1.0]))
    return edit


# ------------------------------------------------------------------------------------------------- each mechanism alone --
ATTENTION_SIZES = [dict(heads=6, dim=64, vdim=56, q_rank=72, kv_rank=112, scale=0.14), dict(heads=3, dim=24, vdim=40, q_rank=20, kv_rank=36, scale=0.4),
                   dict(heads=17, dim=16, vdim=80, q_rank=50, kv_rank=200, scale=0.3), dict(heads=33, dim=100, vdim=128, q_rank=33, kv_rank=64, scale=0.1),
                   dict(heads=1, dim=1, vdim=3, q_rank=2, kv_rank=5, scale=1.0), dict(heads=2, dim=144, vdim=136, q_rank=64, kv_rank=300, scale=0.08),
                   dict(heads=20, dim=128, vdim=64, q_rank=96, kv_rank=512, scale=0.09), dict(heads=2, dim=32, vdim=48, q_rank=40, kv_rank=530, scale=0.2)]


@pytest.mark.parametrize("mix", ATTENTION_SIZES, ids=lambda m: f"{m['heads']}-{m['dim']}-{m['vdim']}-{m['q_rank']}-{m['kv_rank']}")
@DTYPES
def test_latent_attention_alone(mix, dtype):
    raw = raw_config([layer(**mix)], width=72, side=0)
    m, w = build(raw, dtype, edit=only("mix"))
    toks = tokens(210, 61)
    ref = R.forward(raw, w, toks)
    eng = m.step_engine(3, 320)
    assert err(run(eng, 1, 0, toks), ref) < TOL[dtype]
    assert err(run_cut(eng, 2, toks, [190]), ref) < TOL[dtype]                 # the tail through the absorbed form
    assert err(run_cut(eng, 0, toks[:150], [2, 16, 17, 3, 100]), ref[:150]) < TOL[dtype]       # short portions, long ones, behind a past


@pytest.mark.parametrize("ff", [1, 33, 72, 200])
@DTYPES
def test_xielu_feed_forward_alone(ff, dtype):
    raw = raw_config([layer(dense(ff))], width=76, side=0, vocab=203)
    for p, q in ((-3.0, 2.5), (1.5, -4.0)):
        def edit(w):
            only("mlp")(w)
            w["l0.mlp.act"].copy_(torch.tensor([p, q]))
            w["l0.mlp.up"] *= 2
        m, w = build(raw, dtype, edit=edit)
        for T in (1, 40, 130):
            toks = tokens(T, 203, T)
            assert err(run(m.step_engine(1, 256), 0, 0, toks), R.forward(raw, w, toks)) < TOL[dtype], (p, T)


MIXTURES = {"plain": moe(10, 3, 5, (5, 3), 56, 96), "no-identity-no-groups": moe(5, 2, 0, None, 24, 0), "mostly-identity": moe(2, 3, 10, (4, 3), 17, 9),
            "one-of-many": moe(40, 1, 0, (8, 1), 16, 48), "all": moe(3, 4, 1, (2, 2), 40, 0), "one-expert": moe(1, 1, 0, None, 33, 0), "wide-group": moe(70, 9, 58, (2, 1), 8, 8)}


@pytest.mark.parametrize("name", MIXTURES)
@DTYPES
def test_expert_mixture_alone(name, dtype):
    """Few rows (one launch of the router) and many (three), 1 .. 700 tokens."""
    raw = raw_config([layer(MIXTURES[name])], width=68, side=0, vocab=400)
    m, w = build(raw, dtype, edit=only("mlp"))
    eng = m.step_engine(2, 800)
    for T in (1, 2, 17, 40, 64, 65, 300, 700):
        toks = tokens(T, 400, T)
        ref, ok = clear_choices(raw, w, toks) if dtype == BF else (R.forward(raw, w, toks), None)
        if ok is not None:
            assert T < 17 or float(ok.double().mean()) > 0.3
            if not ok.any():
                continue
        assert err(run(eng, 0, 0, toks), ref, ok) < TOL[dtype], T


def test_expert_mixture_in_large_blocks():
    """Enough rows per expert for the 256-row tiles, more than one split of the output product for few rows."""
    raw = raw_config([layer(moe(3, 2, 1, (2, 2), 600, 0))], width=512, side=0, vocab=300)
    m, w = build(raw, BF, edit=only("mlp"))
    eng = m.step_engine(1, 1000)
    for T in (900, 12):
        toks = tokens(T, 300, T)
        ref, ok = clear_choices(raw, w, toks)
        assert err(run(eng, 0, 0, toks), ref, ok) < TOL[BF]


@DTYPES
def test_router_details_show(dtype):
    """Corrections move the choice but not the weights; members of other groups stay out although every choice score is negative; identity experts
    pass their input on.  Each mistake, planted in the restatement, is far outside the tolerance."""
    mlp = moe(9, 3, 3, (4, 2), 32, 0)
    raw = raw_config([layer(mlp)], width=64, side=0, vocab=200)

    def edit(w):
        only("mlp")(w)
        w["l0.mlp.correction"].copy_(torch.linspace(-0.9, -0.5, 12)[torch.randperm(12, generator=torch.Generator().manual_seed(3))])
    m, w = build(raw, dtype, edit=edit)
    toks = tokens(60, 200, 1)
    ref, ok = clear_choices(raw, w, toks)
    assert float(ok.double().mean()) > 0.5
    got = run(m.step_engine(1, 64), 0, 0, toks)
    assert err(got, ref, ok) < TOL[dtype]

    def wrong(**router):
        r2 = dict(raw, layers=[layer(dict(mlp, router=dict(mlp["router"], **router)))])
        return R.forward(r2, w, toks)
    w_nc = dict(w)
    w_nc["l0.mlp.correction"] = torch.zeros(12)
    zero_mask = R.choose

    def masked_to_zero(s, c, router):
        choice, size = (s + c), 3
        best = choice.view(4, 3).max(-1).values.argsort(descending=True)[:2].tolist()
        choice = torch.tensor([float(choice[i]) if i // size in best else 0.0 for i in range(12)])
        return choice.argsort(descending=True)[:3].tolist()
    R.choose = masked_to_zero
    planted = [R.forward(raw, w, toks)]
    R.choose = zero_mask
    planted += [wrong(groups=None), R.forward(raw, w_nc, toks), wrong(top=2)]
    for i, bad in enumerate(planted):
        assert err(bad, ref, ok) > 2 * TOL[dtype], i


@DTYPES
def test_embedding_alone(dtype):
    """Scale and bigram rows; the previous token comes from the slot when a portion or a decoded token starts behind it."""
    raw = raw_config([layer(None)], width=50, vocab=90, scale=2.25, bigram=(31, 5000000029, 77777))

    def edit(w):
        only()(w)
    m, w = build(raw, dtype, edit=edit)
    toks = tokens(90, 90, 4)
    ref = R.forward(raw, w, toks)
    eng = m.step_engine(2, 100)
    for cuts in ([90], [1, 2, 3, 50, 17], [64, 2, 24], []):
        assert err(run_cut(eng, 1, toks, cuts), ref) < TOL[dtype], cuts
    other = tokens(40, 90, 5)                                                  # the slot again: the first token's row does not look back
    assert err(run_cut(eng, 1, other, [30]), R.forward(raw, w, other)) < TOL[dtype]
    swapped = R.forward(dict(raw, embedding=dict(raw["embedding"], bigram=dict(buckets=31, mul_prev=77777, mul_cur=5000000029))), w, toks)
    assert err(swapped, ref) > 0.2


@pytest.mark.parametrize("side", [1, 16, 40, 100])
@DTYPES
def test_token_input_and_depth_average(side, dtype):
    """Two layers with nothing but the token input (their own columns of the table), then strong depth weights; the stream after every layer."""
    raw = raw_config([layer(None), layer(None), layer(None)], width=60, side=side, vocab=70)

    def edit(w):
        for i in range(3):
            w[f"l{i}.ls1"].zero_()
            w[f"l{i}.dwa"].copy_(torch.randn(i + 2, generator=torch.Generator().manual_seed(i)))
            w[f"l{i}.side.gate"] *= 2
    m, w = build(raw, dtype, edit=edit)
    toks, col = tokens(80, 70), []
    ref = R.forward(raw, w, toks, collect=col)
    eng = m.step_engine(1, 128)
    _, res = eng.launch([(0, 0, toks)], residuals=True)
    for i, c in enumerate(col):
        assert err(res[i], c) < (0.012 if dtype == BF else 1e-5), i
    assert err(run_cut(eng, 0, toks, [40, 20]), ref) < TOL[dtype]


@DTYPES
def test_one_norm_weight_and_layer_scales(dtype):
    """A large eps, norm weights far from one, layer scales that differ by column."""
    raw = raw_config([layer(dense(48)), layer(moe())], width=64, eps=0.5)

    def edit(w):
        for k in ("l0.norm1", "l0.norm2", "l1.norm1", "l1.norm2", "final.norm"):
            w[k].fill_({"l0.norm1": 2.5, "l0.norm2": 0.3, "l1.norm1": -1.5, "l1.norm2": 3.0, "final.norm": 0.7}[k])
        for k in ("l0.ls1", "l0.ls2", "l1.ls1", "l1.ls2"):
            w[k].copy_(torch.randn(64, generator=torch.Generator().manual_seed(len(k) + ord(k[1]) + ord(k[-1]))))
    m, w = build(raw, dtype, edit=edit)
    toks = tokens(60, 61)
    ref, ok = clear_choices(raw, w, toks)
    assert err(run(m.step_engine(1, 64), 0, 0, toks), ref, ok if dtype == BF else None) < TOL[dtype]


@DTYPES
def test_sequential_layers_of_other_mixers(dtype):
    """The sequential form is not tied to latent attention: sigmoid attention and a state-space mixer with norms on both sides of every sublayer, a plain
    gated feed-forward, a mixture behind a norm whose identity experts return the NORMED input, a residual multiplier."""
    from onebit_amd.hybrid import ExpertMixture, GatedFeedForward, HybridDecoder, HybridLayer, SigmoidAttention, StateSpace
    g = torch.Generator().manual_seed(5)
    r = lambda *s: torch.randn(*s, generator=g).to(BF)
    lin = lambda n, k: (torch.randn(n, k, generator=g) / k ** 0.5).to(BF)
    W, V, eps, mult = 56, 70, 1e-3, 0.6
    near1 = lambda n: (1 + 0.2 * torch.randn(n, generator=g)).to(BF)
    gate = lambda ff: (lin(ff, W), lin(ff, W), lin(W, ff))
    att = dict(q=lin(4 * 16, W), k=lin(2 * 16, W), v=lin(2 * 24, W), o=lin(W, 4 * 24))
    H, G, N, P, taps = 4, 2, 16, 12, 3
    ssm = dict(w_in=lin(2 * H * P + 2 * G * N + H, W), conv_w=r(H * P + 2 * G * N, taps), conv_b=r(H * P + 2 * G * N), dt_bias=r(H) - 1, A_log=r(H), D=r(H), norm=near1(H * P), o=lin(W, H * P))
    norms = [near1(W) for _ in range(8)]
    ff0, shared, experts = gate(40), gate(24), [gate(20) for _ in range(3)]
    router, corr = (3 * torch.randn(4, W, generator=g) / W ** 0.5).to(BF), r(4) * 0.1
    embed, head, fin = r(V, W), lin(V, W), near1(W)
    cu = lambda t: t.cuda()
    gf = lambda t: GatedFeedForward(*map(cu, t))
    layers = [HybridLayer(cu(norms[0]), SigmoidAttention(4, 2, 16, 24, 0.4, *(cu(att[k]) for k in "qkvo")), gf(ff0), sequential=True, mixer_out=cu(norms[1]),
                          mlp_norm=cu(norms[2]), mlp_out=cu(norms[3])),
              HybridLayer(cu(norms[4]), StateSpace(H, G, N, P, 2, *(cu(ssm[k]) for k in ("w_in", "conv_w", "conv_b", "dt_bias", "A_log", "D", "norm", "o"))),
                          ExpertMixture([gf(e) for e in experts], cu(router), cu(corr), 2, 1, shared=gf(shared)), sequential=True, mlp_norm=cu(norms[5]), mlp_out=cu(norms[6]))]
    m = HybridDecoder(layers=layers, runs=[(0, False), (1, False)], embed=cu(embed), pos_embed=None, final_norm=cu(fin), head=cu(head), eps=eps, residual_mult=mult, dtype=dtype)

    toks = tokens(70, V, 2)
    d = lambda t: t.double()
    nrm = lambda x, w: R.rms(x, eps) * d(w)
    ffn = lambda h, t: R.linear(R.silu(R.linear(h, d(t[0]))) * R.linear(h, d(t[1])), d(t[2]))
    x = d(embed)[torch.tensor(toks)]
    h = nrm(x, norms[0])
    z4 = torch.zeros(4, dtype=torch.float64)
    proj = lambda k, n: R.linear(h, d(att[k])).view(len(toks), n, -1)
    a = lebepel_ref.sigmoid_attention(proj("q", 4), proj("k", 2), proj("v", 2), 0.4, z4, z4, z4, eps)
    x = x + mult * nrm(R.linear(a.reshape(len(toks), -1), d(att["o"])), norms[1])
    x = x + mult * nrm(ffn(nrm(x, norms[2]), ff0), norms[3])
    w = {"in": ssm["w_in"], "conv": ssm["conv_w"], "conv.b": ssm["conv_b"], "dt_bias": ssm["dt_bias"], "A_log": ssm["A_log"], "D": ssm["D"], "norm": ssm["norm"], "o": ssm["o"]}
    x = x + mult * lebepel_ref.mamba2(nrm(x, norms[4]), {k: d(v) for k, v in w.items()}, "", dict(heads=H, groups=G, state=N, vdim=P, norm_groups=2), eps)
    h = nrm(x, norms[5])
    s = torch.softmax(R.linear(h, d(router)), -1)
    y, ok = ffn(h, shared), []
    for t in range(len(toks)):
        order = (s[t] + d(corr)).argsort(descending=True).tolist()
        ok.append(float(s[t, order[1]] + corr[order[1]] - s[t, order[2]] - corr[order[2]]) > 0.02)
        for i in order[:2]:
            y[t] += s[t, i] * (h[t] if i == 3 else ffn(h[t], experts[i]))
    x = x + mult * nrm(y, norms[6])
    ref = R.linear(nrm(x, fin), d(head))
    ok = torch.tensor(ok)
    eng = m.step_engine(2, 80)
    assert float(ok.double().mean()) > 0.6
    assert err(run(eng, 0, 0, toks), ref, ok) < TOL[dtype]
    assert err(run_cut(eng, 1, toks, [50, 2]), ref, ok) < TOL[dtype]


# ------------------------------------------------------------------------------------------------------ whole models --
MODELS = {
    "mixed": raw_config([layer(dense(56)), layer(moe(9, 2, 1, (5, 3), 24, 40)), layer(moe(5, 2, 1, (3, 2), 40, 0), heads=2, dim=32, vdim=48, kv_rank=70)], width=64, vocab=150),
    "odd": raw_config([layer(moe(3, 1, 2, None, 11, 13), heads=5, dim=9, vdim=7, q_rank=13, kv_rank=21, scale=0.6), layer(None), layer(dense(29), heads=1, dim=70, vdim=90, kv_rank=130)],
                      width=50, vocab=77, side=29, bigram=(11, 2, 3)),
    "bare": raw_config([layer(dense(40)), layer(dense(24), heads=4, dim=64, vdim=32, q_rank=48, kv_rank=96, scale=0.1)], width=80, vocab=90, side=0, bigram=None),
}


@pytest.fixture(scope="module")
def zoo():
    """Per (model, dtype): the packed model, a 330-token sequence, its reference logits and the positions that are compared."""
    cache = {}

    def get(name, dtype):
        if (name, dtype) not in cache:
            raw = MODELS[name]
            m, w = build(raw, dtype, seed=5)
            key = ("ref", name)
            if key not in cache:
                toks = tokens(330, raw["vocab"], 9)
                cache[key] = (toks,) + clear_choices(raw, w, toks)
            toks, ref, ok = cache[key]
            if dtype == F32:
                _, ok = ref, torch.ones_like(ok)
            assert float(ok.double().mean()) > 0.7
            cache[(name, dtype)] = (m, toks, ref, ok)
        return cache[(name, dtype)]
    return get


@pytest.mark.parametrize("name", MODELS)
@DTYPES
def test_prompt_against_reference(zoo, name, dtype):
    m, toks, ref, ok = zoo(name, dtype)
    eng = m.step_engine(2, 400)
    assert err(run(eng, 0, 0, toks), ref, ok) < TOL[dtype]
    for n in (1, 2, 3, 15, 16, 17, 63, 64, 65, 127, 128, 129):
        assert err(run(eng, 1, 0, toks[:n]), ref[:n], ok[:n]) < TOL[dtype], n


@pytest.mark.parametrize("name", MODELS)
@DTYPES
def test_portions_and_token_by_token(zoo, name, dtype):
    m, toks, ref, ok = zoo(name, dtype)
    eng = m.step_engine(2, 400)
    assert err(run_cut(eng, 0, toks[:140], []), ref[:140], ok[:140]) < TOL[dtype]              # every token decoded
    assert eng.graph_launches >= 140
    for cuts in ([2] * 70, [3, 61, 64, 2], [129, 65, 127], [1, 2, 128, 1, 64, 60], [200, 2, 2, 90], [16, 17, 15, 32, 18]):
        n = sum(cuts) + 6
        assert err(run_cut(eng, 1, toks[:n], cuts), ref[:n], ok[:n]) < TOL[dtype], cuts


@pytest.mark.parametrize("name", ["mixed", "odd"])
@DTYPES
def test_unequal_batches_and_slot_reuse(zoo, name, dtype):
    """Requests of different lengths entering together, decoding together, mixed with a new prompt: each as if alone; slots freed and used
    again by shorter and longer requests."""
    m, toks, ref, ok = zoo(name, dtype)
    eng = m.step_engine(4, 400)
    for lens in ((5, 130, 1, 67), (300, 2, 64, 9)):                              # second round: every slot used before
        out = [[] for _ in lens]
        eng.launch([(s, 0, toks[:n], list(range(n))) for s, n in enumerate(lens)])
        lg, at = eng.logits[:sum(lens)].clone(), 0
        for s, n in enumerate(lens):
            out[s].append(lg[at:at + n])
            at += n
        pos = list(lens)
        for k in range(8):
            live = [s for s in (3, 1, 0, 2) if not (s == 1 and k >= 5)]          # one ends early; the order of items is free
            eng.launch([(s, pos[s], toks[pos[s]:pos[s] + 1]) for s in live])
            for i, s in enumerate(live):
                out[s].append(eng.logits[i:i + 1].clone())
                pos[s] += 1
        # slot 1 is given to another request whose prompt shares a step with the others' next tokens, a short portion and a longer one
        eng.launch([(0, pos[0], toks[pos[0]:pos[0] + 1]), (1, 0, toks[:21], list(range(21))), (3, pos[3], toks[pos[3]:pos[3] + 3], [0, 2]),
                    (2, pos[2], toks[pos[2]:pos[2] + 18], [17])])
        mixed = eng.logits[:25].clone()
        for s, n in enumerate(lens):
            got = torch.cat(out[s])
            assert err(got, ref[:got.shape[0]], ok[:got.shape[0]]) < TOL[dtype], (lens, s)
        at = [pos[0]] + list(range(21)) + [pos[3], pos[3] + 2, pos[2] + 17]
        assert err(mixed, ref[at], ok[at]) < TOL[dtype]


@DTYPES
def test_many_requests_and_expansion_in_groups(zoo, dtype):
    """70 prompts in one step (more than one table of segments), then portions behind long pasts whose keys do not all fit the expansion buffer."""
    m, toks, ref, ok = zoo("mixed", dtype)
    eng = m.step_engine(72, 64, max_rows=64)
    lens = [17 + i % 5 for i in range(70)]
    eng.launch([(s, 0, toks[:n], [n - 1]) for s, n in enumerate(lens)])
    at = [n - 1 for n in lens]
    assert err(eng.logits[:70], ref[at], ok[at]) < TOL[dtype]
    eng.launch([(s, n, toks[n:n + 1]) for s, n in enumerate(lens)])              # 70 single tokens in one graph
    assert err(eng.logits[:70], ref[lens], ok[lens]) < TOL[dtype]
    eng = m.step_engine(6, 1000, max_rows=64)
    far = (toks * 4)[:960]
    for s in range(6):
        eng.launch([(s, 0, far[:900 + s])])
    alone = []
    for s in range(6):
        alone.append(run(eng, s, 900 + s, far[900 + s:925 + s]))
    eng.launch([(s, 900 + s, far[900 + s:925 + s], list(range(25))) for s in range(6)])
    assert err(eng.logits[:150], torch.cat(alone).cpu()) < (0.02 if dtype == BF else 1e-5)


@pytest.mark.parametrize("seed", range(6))
def test_random_sizes(seed):
    """Layers of random kinds and sizes in fp32: whole, and in random portions."""
    import random
    rg = random.Random(seed)

    def lay():
        m = dict(heads=rg.randint(1, 20), dim=rg.choice([8, 12, 24, 48, 80, 136]), vdim=rg.choice([8, 20, 32, 72, 96, 144]), q_rank=rg.choice([17, 32, 60, 96]),
                 kv_rank=rg.choice([24, 50, 96, 160, 256, 520]))
        kind = rg.randrange(3)
        if kind == 0:
            return layer(None if rg.random() < 0.3 else dense(rg.choice([7, 32, 100])), scale=m["dim"] ** -0.5, **m)
        experts, identity = rg.randint(2, 20), rg.choice([0, 1, 4, 6])
        counts = [c for c in range(1, experts + identity) if (experts + identity) % c == 0]
        count = rg.choice(counts)
        keep = rg.randint(1, count)
        return layer(moe(experts, rg.randint(1, min(6, keep * ((experts + identity) // count))), identity, (count, keep), rg.choice([8, 17, 64]), rg.choice([0, 24, 100])),
                     scale=m["dim"] ** -0.5, **m)
    raw = raw_config([lay() for _ in range(rg.randint(1, 4))], width=rg.choice([48, 50, 100, 192]), vocab=rg.choice([61, 100, 300]), side=rg.choice([0, 18, 33]),
                     bigram=rg.choice([None, (101, 19, 11)]))
    m, w = build(raw, F32, seed=seed)
    toks = tokens(150, raw["vocab"], seed)
    ref, eng, cuts = R.forward(raw, w, toks), m.step_engine(3, 200), []
    while sum(cuts) < 140:
        cuts.append(min(142 - sum(cuts), rg.choice([1, 2, 5, 16, 17, 40, 64])))
    assert err(run(eng, 0, 0, toks), ref) < TOL[F32] and err(run_cut(eng, 1, toks, cuts), ref) < TOL[F32], (raw, cuts)


@DTYPES
def test_does_not_depend_on_batch_or_slots(zoo, dtype):
    """The same request alone and in company: equal up to the rounding of the work type (both against the reference is not enough)."""
    m, toks, _, ok = zoo("mixed", dtype)
    eng = m.step_engine(8, 400)
    alone = run_cut(eng, 0, toks[:100], [90])
    eng.launch([(s, 0, toks[s:s + 20 + 13 * s]) for s in range(7)] + [(7, 0, toks[:90], list(range(90)))])
    got = [eng.logits[7:97].clone()]
    for t in range(90, 100):
        eng.launch([(7, t, toks[t:t + 1])] + [(s, 20 + 13 * s + t - 90, [3]) for s in range(7)])
        got.append(eng.logits[:1].clone())
    assert err(torch.cat(got), alone.cpu(), ok[:100]) < (0.02 if dtype == BF else 1e-5)


@DTYPES
def test_growing_slots_keeps_live_requests(zoo, dtype):
    m, toks, ref, ok = zoo("mixed", dtype)
    eng = m.step_engine(2, 400)
    eng.launch([(0, 0, toks[:50]), (1, 0, toks[:20])])
    eng.grow(5)
    assert eng.n_slots == 5
    eng.launch([(4, 0, toks[:33], [32]), (0, 50, toks[50:51]), (1, 20, toks[20:22], [0, 1])])
    at = [32, 50, 20, 21]
    assert err(eng.logits[:4], ref[at], ok[at]) < TOL[dtype]


# ------------------------------------------------------------------------------------- far keys: one score that stands out --
def far_model(dtype, dim, kv_rank, heads=2):
    """One layer, attention alone, in which token 1 asks for token 0's key: its score stands out by about 12 against scores near zero."""
    raw = raw_config([layer(heads=heads, dim=dim, vdim=dim, q_rank=8, kv_rank=kv_rank, scale=1.0)], width=64, vocab=40, scale=1.0, bigram=None, side=0)

    def edit(w):
        g = torch.Generator().manual_seed(2)
        only("mix")(w)
        w["embed"].copy_(torch.nn.functional.one_hot(torch.arange(40), 64).to(BF) * 4)
        for n in ("dq", "dkv", "uq", "uk"):
            w["l0.mix." + n].zero_()
        w["l0.mix.dq.norm"].fill_(1.0), w["l0.mix.dkv.norm"].fill_(1.0)
        # every token's query latent is one direction, token 1's another; likewise the key latents, token 0's own; the rest spread for the values
        w["l0.mix.dq"][0, :40], w["l0.mix.dq"][0, 1], w["l0.mix.dq"][1, 1] = 1.0, 0.0, 1.0
        w["l0.mix.dkv"][1:, 2:40] = torch.randn(kv_rank - 1, 38, generator=g).to(BF)
        w["l0.mix.dkv"][0, 0] = 1.0
        key = torch.randn(dim, generator=g)
        key = key * (12.0 / (key.norm() ** 2 * 8 ** 0.5 * kv_rank ** 0.5)) ** 0.5
        for h in range(heads):
            w["l0.mix.uq"][h * dim:(h + 1) * dim, 1] = key.to(BF)
            w["l0.mix.uk"][h * dim:(h + 1) * dim, 0] = key.to(BF)
    m, w = build(raw, dtype, seed=1, edit=edit)
    return raw, m, w


def last_logits(raw, w, toks, drop=None, twice=None):
    """Reference logits of the last position only; ``drop`` / ``twice``: plant the mistake of losing or doubling that key."""
    w = {k: v.double() for k, v in w.items()}
    mix, eps = raw["layers"][0]["mixer"], raw["norm"]["eps"]
    H, p = mix["heads"], "l0.mix."
    x = R.embedding(raw, w, toks)
    q = R.linear(R.rms(R.linear(x[-1:], w[p + "dq"]), eps) * w[p + "dq.norm"], w[p + "uq"]).view(H, -1)
    c = R.rms(R.linear(x, w[p + "dkv"]), eps) * w[p + "dkv.norm"]
    k, v = R.linear(c, w[p + "uk"]).view(len(toks), H, -1), R.linear(c, w[p + "uv"]).view(len(toks), H, -1)
    o = []
    for h in range(H):
        a = torch.exp((k[:, h] @ q[h]) * mix["scale"])
        if drop is not None:
            a[drop] = 0
        if twice is not None:
            a[twice] *= 2
        o.append(a @ v[:, h] / a.sum())
    y = R.linear(torch.cat(o)[None], w[p + "o"])
    y = x[-1:] + R.rms(y, eps) * w["l0.norm1"] * w["l0.ls1"]
    return R.linear(R.rms(y, eps) * w["final.norm"], w["head"])[0]


@pytest.mark.parametrize("dim,kv_rank", [(32, 40), (64, 128), (128, 250), (160, 64), (96, 512), (48, 600)])
@DTYPES
def test_far_keys_in_prompts_and_decoding(dim, kv_rank, dtype):
    """The asked-for token at the edges of the kernels' bands, key blocks, query blocks and context splits, as prompt, as a short portion and decoded.
    A lost key in the restatement is far outside the tolerance."""
    raw, m, w = far_model(dtype, dim, kv_rank, heads=17 if kv_rank == 250 else 2)
    eng = m.step_engine(3, 1300)
    base = torch.randint(2, 40, (1200,), generator=torch.Generator().manual_seed(0)).tolist()
    for n, places in ((130, (0, 1, 15, 16, 62, 63, 64, 65, 127, 128)), (700, (0, 63, 255, 256, 511, 512, 640, 698)), (1200, (0, 127, 128, 1023, 1024, 1150))):
        for far in places:
            toks = list(base[:n])
            toks[far], toks[n - 1] = 0, 1
            ref, lost = last_logits(raw, w, toks), last_logits(raw, w, toks, drop=far)
            scale = float(ref.pow(2).mean().sqrt())
            assert float((ref - lost).pow(2).mean().sqrt()) / scale > 0.15, "the far key does not show"
            eng.launch([(0, 0, toks)])                                           # in the prompt
            p = eng.logits[0].double().cpu()
            eng.launch([(1, 0, toks[:-1])])                                      # decoded
            eng.launch([(1, n - 1, toks[-1:])])
            d = eng.logits[0].double().cpu()
            eng.launch([(2, 0, toks[:-2])])                                      # the last two as a portion
            eng.launch([(2, n - 2, toks[-2:])])
            s = eng.logits[0].double().cpu()
            for got, what in ((p, "prompt"), (d, "decoded"), (s, "portion")):
                assert float((got - ref).pow(2).mean().sqrt()) / scale < TOL[dtype], (dim, n, far, what)


@DTYPES
def test_first_tokens_and_visible_edge(dtype):
    """The newest key is visible to its own token and to nobody before it; the first token sees itself alone."""
    raw, m, w = far_model(dtype, 64, 100)
    eng = m.step_engine(2, 300)
    base = torch.randint(2, 40, (200,), generator=torch.Generator().manual_seed(7)).tolist()
    for at in (0, 1, 15, 16, 63, 64, 127, 128, 190):
        toks = list(base)
        toks[at] = 1                                                            # asks; the key it asks for comes right after it
        toks[at + 1] = 0
        ref = last_logits(raw, w, toks[:at + 1])
        scale = float(ref.pow(2).mean().sqrt())
        eng.launch([(0, 0, toks, [at])])
        assert float((eng.logits[0].double().cpu() - ref).pow(2).mean().sqrt()) / scale < TOL[dtype], at
        saw = last_logits(raw, w, toks[:at] + [0, 1])                           # (what it would be with that key in sight)
        assert float((saw - ref).pow(2).mean().sqrt()) / scale > 0.15


def test_long_decoding_stays_exact():
    """600 decoded tokens in fp32 and bf16 against whole prompts of the same kernels' fp32 form."""
    raw = MODELS["bare"]
    m32, _ = build(raw, F32, seed=8)
    m16, _ = build(raw, BF, seed=8)
    toks = tokens(640, raw["vocab"], 4)
    e32, e16 = m32.step_engine(2, 640), m16.step_engine(2, 640)
    whole = run(e32, 0, 0, toks)
    assert err(run_cut(e32, 1, toks, [40])[-100:], whole[-100:].cpu()) < 2e-5
    assert err(run_cut(e16, 1, toks, [40])[-100:], whole[-100:].cpu()) < TOL[BF]


@DTYPES
def test_graph_replays_equal_eager_steps(zoo, dtype):
    """Every replay of a single-token step equals the step launched directly, with other work between the replays."""
    m, toks, _, _ = zoo("mixed", dtype)
    a, b = m.step_engine(3, 400), m.step_engine(3, 400, use_graph=False)
    for e in (a, b):
        e.launch([(s, 0, toks[s:40 + s]) for s in range(3)])
    for t in range(30):
        items = [(s, 40 + t, toks[40 + s + t:41 + s + t]) for s in ((0, 2, 1) if t % 3 else (1, 2))]
        items = [(s, p if (s != 0) else 40 + t - (t + 2) // 3, k) for s, p, k in items]
        na, nb = a.launch(items).clone(), b.launch(items).clone()
        la, lb = a.logits[:len(items)].clone(), b.logits[:len(items)].clone()
        _ = torch.randn(1000, 1000, device="cuda") @ torch.randn(1000, 1000, device="cuda")
        torch.cuda.synchronize()
        assert torch.equal(na, nb) and torch.equal(la, lb), t
        if t % 7 == 3:
            a.launch([(2, 0, toks[:25])]), b.launch([(2, 0, toks[:25])])         # a prompt between replays; slot 2 starts over
            a.launch([(2, 25, toks[25:41 + t])]), b.launch([(2, 25, toks[25:41 + t])])
    assert a.graph_launches == 30 and b.graph_launches == 0


# ------------------------------------------------------------------------------------------- the framework's entry points --
def greedy_reference(raw, w, prompt, n):
    out, gaps = list(prompt), []
    for _ in range(n):
        top = R.forward(raw, w, out)[-1].topk(2)
        gaps.append(float(top.values[0] - top.values[1]))
        out.append(int(top.indices[0]))
    return out[len(prompt):], gaps


@pytest.mark.parametrize("chunk", [None, 5, 2])
def test_greedy_generation_through_the_scheduler(chunk):
    from onebit_amd.serving import ContinuousBatcher
    raw = raw_config([layer(dense()), layer(moe())], width=64, vocab=50)
    m, w = build(raw, F32, seed=11)
    prompts = [tokens(n, 50, n) for n in (3, 17, 1, 9, 26)]
    cb = ContinuousBatcher(m, max_batch=2, max_len=60, prefill_chunk=chunk)      # fewer slots than requests
    ids = [cb.add_request(p, 6) for p in prompts]
    out = cb.run()
    for i, p in zip(ids, prompts):
        want, gaps = greedy_reference(raw, w, p, 6)
        n = next((k for k, gp in enumerate(gaps) if gp < 1e-4), 6)
        assert out[i][:n] == want[:n] and n >= 1, (p, out[i], want)
    assert cb.graph_steps > 0 and cb.mixed_steps > 0 and cb.steps == cb.graph_steps + cb.mixed_steps


def test_generate_forward_and_evaluation_callers():
    from onebit_amd.evaluate import loglikelihood_tokens, perplexity
    raw = raw_config([layer(moe()), layer(dense())], width=64, vocab=50)
    m, w = build(raw, F32, seed=2)
    ids = torch.tensor([tokens(7, 50, 1), tokens(7, 50, 2)])
    lg = m(ids.cuda())
    ref = torch.stack([R.forward(raw, w, r) for r in ids.tolist()])
    assert err(lg.view(14, -1), ref.view(14, -1)) < TOL[F32]
    out = m.generate(ids, 5)
    assert out.shape == (2, 12) and torch.equal(out[:, :7].cpu(), ids)
    for r, row in zip(ids.tolist(), out.tolist()):
        assert row[7] == int(R.forward(raw, w, r)[-1].argmax())
    seq = tokens(60, 50, 5)
    want = torch.stack([torch.log_softmax(R.forward(raw, w, seq[i:i + 20]), -1)[:-1].gather(1, torch.tensor(seq[i + 1:i + 20])[:, None]).mean() for i in (0, 20, 40)])
    assert abs(perplexity(m, torch.tensor([seq]), 20) / float(torch.exp(-want.mean())) - 1) < 1e-3
    reqs = [(seq[:10], seq[10:14]), (seq[:3], seq[3:5]), (seq[20:45], seq[45:46])]
    for (c, t), (lp, _) in zip(reqs, loglikelihood_tokens(m, reqs, 2, 64)):
        full = torch.log_softmax(R.forward(raw, w, list(c) + list(t)), -1)
        assert abs(lp - sum(float(full[len(c) - 1 + i, tok]) for i, tok in enumerate(t))) < 1e-3


def test_model_folder_trace_and_command_line(tmp_path, capsys):
    import io
    from onebit_amd.checkpoint import write_safetensors
    from onebit_amd.cli import main
    from onebit_amd.trace import run as trace_run
    raw = raw_config([layer(dense()), layer(dense(24), heads=2, dim=40)], width=64, vocab=50)
    w = synthetic_weights(SerotarConfig.from_dict(raw), 6)
    (tmp_path / "config.json").write_text(json.dumps(raw))
    write_safetensors(str(tmp_path / "model.safetensors"), w)
    a, b = tokens(12, 50, 1), tokens(31, 50, 2)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:9], "want": [0, 8]}, {"id": "b", "tokens": b[:30], "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[9:10], "want": []}, {"id": "b", "tokens": b[30:], "want": [0]}], "end": ["b"]},
             {"step": 2, "entries": [{"id": "a", "tokens": a[10:], "want": [1]}], "end": ["a"]},
             {"step": 3, "entries": [{"id": "c", "tokens": b[:5], "want": [4]}], "end": ["c"]}]
    ra, rb = R.forward(raw, w, a), R.forward(raw, w, b)
    for dtype, tol in (("bfloat16", TOL[BF]), ("float32", TOL[F32])):
        out = tmp_path / dtype
        assert trace_run(str(tmp_path), dtype, str(out), 64, lines=io.StringIO("\n".join(json.dumps(s) for s in steps))) == 0
        assert [l for l in capsys.readouterr().out.splitlines() if l.startswith("done")] == [f"done {i}" for i in range(4)]
        load = lambda i: torch.frombuffer(bytearray((out / f"{i}.f32").read_bytes()), dtype=torch.float32).view(-1, 50)
        assert err(load(0), ra[[0, 8]]) < tol and err(load(1), rb[[30]]) < tol and err(load(2), ra[[11]]) < tol and err(load(3), rb[[4]]) < tol
    assert main(["generate", "--model", str(tmp_path), "--dtype", "float32", "--prompt", ",".join(map(str, a)), "--prompt", "3 4", "--max-new-tokens", "3"]) == 0
    rows = [json.loads(l) for l in capsys.readouterr().out.splitlines() if l.startswith("{")]
    assert len(rows) == 2 and rows[0]["tokens"][0] == int(ra[-1].argmax())


def test_launch_errors(zoo):
    m, toks, _, _ = zoo("bare", F32)
    eng = m.step_engine(2, 100)
    for items in ([(2, 0, [1])], [(0, 0, [1]), (0, 0, [2])], [(0, 98, [1, 2, 3])], [(0, 0, [90])], [(0, 0, [1, -1])], [(0, 0, [1, 2], [2])], []):
        with pytest.raises(ValueError):
            eng.launch(items)
