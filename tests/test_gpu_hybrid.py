"""Hybrid decoders on the GPU against the plain restatement (oracle/lebepel_ref.py, float64): each mechanism alone, prompts, decoding through the
cache and state, portions, batches, slots used again, far keys, odd sizes, generation through the scheduler.

Weights are random bf16, so the restatement runs on the very numbers the kernels read; what remains is the rounding of bf16 activations
(``TOL``), or fp32 rounding."""
import json

import pytest
import torch

from onebit_amd.lebepel import LebepelConfig, LebepelForCausalLM, synthetic_weights
from oracle import lebepel_ref as R
from test_hybrid_cpu import att, raw_config, ssm

pytestmark = pytest.mark.gpu
BF, F32 = torch.bfloat16, torch.float32
TOL = {BF: 0.03, F32: 3e-5}
DTYPES = pytest.mark.parametrize("dtype", [BF, F32], ids=["bf16", "f32"])


def build(raw, dtype, seed=0, edit=None):
    cfg = LebepelConfig.from_dict(raw)
    w = synthetic_weights(cfg, seed)
    if edit is not None:
        edit(w)
    return LebepelForCausalLM(cfg, w, dtype), w


def tokens(n, vocab, seed=0):
    return torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def err(got, want):
    """The largest row error: rms of the difference over the rms of the whole reference."""
    got, want = got.double().cpu(), want.double()
    return float(((got - want).pow(2).mean(-1).sqrt() / want.pow(2).mean().sqrt()).max())


def run(eng, slot, start, toks):
    """Logits of every row of one portion, as the host sees them."""
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


# ------------------------------------------------------------------------------------------------- each mechanism alone --
@pytest.mark.parametrize("T", [1, 7, 16, 17, 33, 64, 65, 130, 300])
@DTYPES
def test_dense_product(T, dtype):
    from onebit_amd import _lib
    from onebit_amd.hybrid import k_tile, pack_fragments
    lib = _lib.load_hybrid()
    g = torch.Generator(device="cuda").manual_seed(T)
    for N, nkt, splits in ((16, 1, (1,)), (80, 6, (1, 2, 3)), (272, 24, (1, 4, 8))):
        K = nkt * k_tile(dtype)
        w, a = torch.randn(N, K, generator=g, device="cuda").to(dtype), torch.randn(T, K, generator=g, device="cuda").to(dtype)
        wp, ap = pack_fragments(w, dtype), torch.zeros(256 * -(-T // 256) // 16, nkt, 64, k_tile(dtype) // 4, dtype=dtype, device="cuda")
        ap[:-(-T // 16)] = pack_fragments(a, dtype)
        ref = a.double() @ w.double().t()
        for s in splits:
            z = torch.full((s, T, N), float("nan"), device="cuda")
            _lib.check_hybrid(lib.onebit_hybrid_gemm(wp.data_ptr(), ap.data_ptr(), z.data_ptr(), 2 if dtype == BF else 1, N // 16, nkt, T, s,
                                                     torch.cuda.current_stream().cuda_stream), "gemm")
            torch.cuda.synchronize()
            assert float((z.double().sum(0) - ref).abs().max()) < 1e-5 * K, (N, nkt, s)


def test_dense_product_large_tiles():
    """The 256 x 256 tiles (enough of them to fill the chip), a ragged last row block and the fp32 accumulation over a long K."""
    from onebit_amd import _lib
    from onebit_amd.hybrid import pack_fragments
    lib = _lib.load_hybrid()
    N, T, K = 4112, 3599, 1568
    w, a = torch.randn(N, K, device="cuda").to(BF), torch.randn(T, K, device="cuda").to(BF)
    wp, ap = pack_fragments(w, BF), torch.zeros(3840 // 16, K // 32, 64, 8, dtype=BF, device="cuda")
    ap[:-(-T // 16)] = pack_fragments(a, BF)
    z = torch.full((T, N), float("nan"), device="cuda")
    _lib.check_hybrid(lib.onebit_hybrid_gemm(wp.data_ptr(), ap.data_ptr(), z.data_ptr(), 2, N // 16, K // 32, T, 1, torch.cuda.current_stream().cuda_stream), "gemm")
    torch.cuda.synchronize()
    ref = a.float() @ w.float().t()
    assert float((z - ref).abs().max()) < 1e-4 * K ** 0.5


ATTENTION_SIZES = [dict(heads=4, kv_heads=4, dim=64, vdim=64, scale=0.125), dict(heads=6, kv_heads=2, dim=24, vdim=40, scale=0.4),
                   dict(heads=8, kv_heads=1, dim=128, vdim=80, scale=0.05), dict(heads=5, kv_heads=5, dim=20, vdim=7, scale=0.7),
                   dict(heads=2, kv_heads=1, dim=144, vdim=136, scale=0.1), dict(heads=1, kv_heads=1, dim=1, vdim=3, scale=1.0),
                   dict(heads=10, kv_heads=2, dim=66, vdim=100, scale=0.2)]


@pytest.mark.parametrize("mix", ATTENTION_SIZES, ids=lambda m: f"{m['heads']}-{m['kv_heads']}-{m['dim']}-{m['vdim']}")
@DTYPES
def test_attention_alone(mix, dtype):
    raw = raw_config([att(**mix, ff=None)], width=72, vocab=61, max_positions=320)
    m, w = build(raw, dtype)
    toks = tokens(210, 61)
    ref = R.forward(raw, w, toks)
    eng = m.step_engine(3, 320)
    assert err(run(eng, 1, 0, toks), ref) < TOL[dtype]
    assert err(run_cut(eng, 2, toks, [190]), ref) < TOL[dtype]                 # the tail through decode attention


SSM_SIZES = [dict(heads=4, groups=2, state=48, vdim=64, conv=4, norm_groups=2), dict(heads=6, groups=1, state=16, vdim=20, conv=2, norm_groups=1),
             dict(heads=3, groups=3, state=100, vdim=33, conv=1, norm_groups=3), dict(heads=2, groups=1, state=128, vdim=64, conv=4, norm_groups=2),
             dict(heads=8, groups=4, state=13, vdim=5, conv=5, norm_groups=4), dict(heads=1, groups=1, state=200, vdim=40, conv=3, norm_groups=1),
             dict(heads=2, groups=2, state=300, vdim=16, conv=7, norm_groups=1)]


@pytest.mark.parametrize("mix", SSM_SIZES, ids=lambda m: f"{m['heads']}-{m['groups']}-{m['state']}-{m['vdim']}-{m['conv']}")
@DTYPES
def test_state_space_alone(mix, dtype):
    raw = raw_config([ssm(**mix, ff=None)], width=72, vocab=61, max_positions=256)
    m, w = build(raw, dtype)
    toks = tokens(150, 61, 1)
    ref = R.forward(raw, w, toks)
    eng = m.step_engine(3, 256)
    assert err(run(eng, 1, 0, toks), ref) < TOL[dtype]
    assert err(run_cut(eng, 2, toks, [64, 2, 61]), ref) < TOL[dtype]           # state and convolution inputs carried over, then decoded


@DTYPES
def test_recurrent_state_is_the_definitions(dtype):
    """The fp32 state a prompt leaves, whatever its length, is the recurrence's (not only its effect on logits)."""
    mix = dict(heads=2, groups=1, state=24, vdim=12, conv=3, norm_groups=1)
    raw = raw_config([ssm(**mix, ff=None)], width=48, vocab=61, max_positions=256)
    m, w = build(raw, dtype)
    w = {k: v.double() for k, v in w.items()}
    for T in (1, 2, 63, 64, 65, 150):
        toks = tokens(T, 61, T)
        h = R.norm(R.embedding(toks, w["embed"], w["pos"]), w["l0.norm1"], raw["norm"]["eps"])
        z, xbc, dt = R.linear(h, w["l0.mix.in"]).split([24, 24 + 48, 2], dim=1)
        x, B, C = R.silu(R.short_conv(xbc, w["l0.mix.conv"], w["l0.mix.conv.b"])).split([24, 24, 24], dim=1)
        _, S = R.ssm(x.reshape(T, 2, 12), B.reshape(T, 1, 24), C.reshape(T, 1, 24), R.softplus(dt + w["l0.mix.dt_bias"]), w["l0.mix.A_log"], w["l0.mix.D"])
        eng = m.step_engine(2, 256)
        eng.launch([(1, 0, toks)])
        got = eng.states.runs[0][0][1][..., :12].double().cpu()
        assert float((got - S).norm() / S.norm()) < (0.01 if dtype == BF else 1e-5), T
        ring = eng.states.runs[0][1][1].double().cpu()
        for t in range(max(0, T - 2), T):                                       # the taps - 1 inputs the next token reads
            assert float((ring[t % 3] - xbc[t]).norm() / xbc[t].norm()) < (0.01 if dtype == BF else 1e-5), (T, t)


@DTYPES
def test_feed_forward_norm_embedding_head_alone(dtype):
    """The mixer silenced (zero output projection): what is left is embedding + positions, the zero-centred norm, the gated
    feed-forward, the residual multiplier, the soft-capped head."""
    raw = raw_config([att(ff=88, heads=2, kv_heads=1)], width=100, vocab=203, mult=0.37, cap=2.0, eps=0.3)

    def silence(w):
        w["l0.mix.o"].zero_(), w["l0.mix.o.b"].zero_()
    m, w = build(raw, dtype, edit=silence)
    toks = tokens(40, 203)
    assert err(run(m.step_engine(1, 64), 0, 0, toks), R.forward(raw, w, toks)) < TOL[dtype]
    # and with the soft cap far away
    raw2 = dict(raw, logit_softcap=1e4)
    m2, _ = build(raw2, dtype, edit=silence)
    assert err(run(m2.step_engine(1, 64), 0, 0, toks), R.forward(raw2, w, toks)) < TOL[dtype]


@DTYPES
def test_residual_stream_after_every_run(dtype):
    """Looped stretch in the middle, a layer without feed-forward before it, one after it: the stream after every run, and the embedding output
    added exactly before later passes."""
    raw = raw_config([ssm(ff=None), att(), ssm(heads=2, groups=1, vdim=12, norm_groups=1), att(ff=33)], loop={"start": 1, "stop": 3, "times": 3}, width=52)
    m, w = build(raw, dtype)
    toks, col = tokens(30, 61), []
    R.forward(raw, w, toks, collect=col)
    _, res = m.step_engine(1, 64).launch([(0, 0, toks)], residuals=True)
    assert res.shape[0] == len(col) == 8
    for i, c in enumerate(col):
        assert err(res[i], c) < (0.01 if dtype == BF else 1e-5), i


# ------------------------------------------------------------------------------------------------------ whole models --
MODELS = {
    "plain": raw_config([ssm(), att()], width=64),
    "looped": raw_config([ssm(heads=4, groups=1, state=40, vdim=24, conv=3), att(heads=4, kv_heads=1, dim=32, vdim=48, scale=0.25), att(dim=64, vdim=16)],
                         loop={"start": 0, "stop": 2, "times": 2}, width=96, vocab=150),
    "odd": raw_config([att(heads=3, kv_heads=3, dim=12, vdim=20, scale=1.1, ff=27), ssm(heads=3, groups=3, state=20, vdim=12, conv=5, norm_groups=1, ff=None)],
                      width=50, vocab=77, mult=1.0, loop={"start": 1, "stop": 2, "times": 2}),
}
for _m in MODELS.values():
    _m["max_positions"] = 1400


@pytest.fixture(scope="module")
def zoo():
    """Per (model, dtype): the packed model, its weights, a 330-token sequence and its reference logits."""
    cache = {}

    def get(name, dtype):
        if (name, dtype) not in cache:
            raw = MODELS[name]
            m, w = build(raw, dtype, seed=5)
            key = ("ref", name)
            if key not in cache:
                toks = tokens(330, raw["vocab"], 9)
                cache[key] = (toks, R.forward(raw, w, toks))
            cache[(name, dtype)] = (m,) + cache[key]
        return cache[(name, dtype)]
    return get


@pytest.mark.parametrize("name", MODELS)
@DTYPES
def test_prompt_against_reference(zoo, name, dtype):
    m, toks, ref = zoo(name, dtype)
    eng = m.step_engine(2, 400)
    assert err(run(eng, 0, 0, toks), ref) < TOL[dtype]
    for n in (1, 2, 3, 63, 64, 65, 127, 128, 129):
        assert err(run(eng, 1, 0, toks[:n]), ref[:n]) < TOL[dtype], n


@pytest.mark.parametrize("name", MODELS)
@DTYPES
def test_portions_and_token_by_token(zoo, name, dtype):
    m, toks, ref = zoo(name, dtype)
    eng = m.step_engine(2, 400)
    assert err(run_cut(eng, 0, toks[:140], []), ref[:140]) < TOL[dtype]         # every token decoded
    assert eng.graph_launches >= 140
    for cuts in ([2] * 70, [3, 61, 64, 2], [129, 65, 127], [1, 2, 128, 1, 64, 60], [200, 2, 2, 90]):
        n = sum(cuts)
        assert err(run_cut(eng, 1, toks[:n + 6], cuts), ref[:n + 6]) < TOL[dtype], cuts


@pytest.mark.parametrize("name", ["looped", "odd"])
@DTYPES
def test_unequal_batches_and_slot_reuse(zoo, name, dtype):
    """Requests of different lengths entering together, decoding together, mixed with a new prompt: each as if alone; slots freed and used
    again by shorter and longer requests."""
    m, toks, ref = zoo(name, dtype)
    eng = m.step_engine(4, 400)
    for lens in ((5, 130, 1, 67), (300, 2, 64, 9)):                              # second round: every slot used before
        out = [[] for _ in lens]
        items = [(s, 0, toks[:n], list(range(n))) for s, n in enumerate(lens)]
        eng.launch(items)
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
        # slot 1 is given to another request whose prompt shares a step with the others' next tokens
        eng.launch([(0, pos[0], toks[pos[0]:pos[0] + 1]), (1, 0, toks[:21], list(range(21))), (3, pos[3], toks[pos[3]:pos[3] + 3], [0, 2])])
        mixed = eng.logits[:24].clone()
        for s, n in enumerate(lens):
            got = torch.cat(out[s])
            assert err(got, ref[:got.shape[0]]) < TOL[dtype], (lens, s)
        assert err(mixed[:1], ref[pos[0]:pos[0] + 1]) < TOL[dtype]
        assert err(mixed[1:22], ref[:21]) < TOL[dtype]
        assert err(mixed[22:], ref[[pos[3], pos[3] + 2]]) < TOL[dtype]


@DTYPES
def test_does_not_depend_on_batch_or_slots(zoo, dtype):
    """The same request alone and in company: equal up to the rounding of the work type (both against the reference is not enough)."""
    m, toks, _ = zoo("looped", dtype)
    eng = m.step_engine(8, 400)
    alone = run_cut(eng, 0, toks[:100], [90])
    eng.launch([(s, 0, toks[s:s + 20 + 13 * s]) for s in range(7)] + [(7, 0, toks[:90], list(range(90)))])
    got = [eng.logits[7:97].clone()]
    for t in range(90, 100):
        eng.launch([(7, t, toks[t:t + 1])] + [(s, 20 + 13 * s + t - 90, [3]) for s in range(7)])
        got.append(eng.logits[:1].clone())
    assert err(torch.cat(got), alone.cpu()) < (0.02 if dtype == BF else 1e-5)


@DTYPES
def test_growing_slots_keeps_live_requests(zoo, dtype):
    m, toks, ref = zoo("plain", dtype)
    eng = m.step_engine(2, 400)
    eng.launch([(0, 0, toks[:50]), (1, 0, toks[:20])])
    eng.grow(5)
    assert eng.n_slots == 5
    eng.launch([(4, 0, toks[:33], [32]), (0, 50, toks[50:51]), (1, 20, toks[20:22], [0, 1])])
    assert err(eng.logits[:4], ref[[32, 50, 20, 21]]) < TOL[dtype]


# ------------------------------------------------------------------------------------- far keys: one score that stands out --
def far_model(dtype, dim, scale=0.5, pb=-9.0, heads=2, kv_heads=1, G=None):
    """Attention whose visible weights are all but zero (pb) except between one token A and one token B: unit-RMS key of A and query of B are
    the same vector.  Position vectors are zero, so only the distance bias sees positions."""
    raw = raw_config([att(heads=heads, kv_heads=kv_heads, dim=dim, vdim=dim, scale=scale, ff=None)], width=64, vocab=40, max_positions=1400, mult=1.0, cap=50.0)

    def edit(w):
        w["pos"].zero_()
        for b in ("q.b", "k.b", "v.b"):
            w["l0.mix." + b].zero_()
        w["embed"].copy_(torch.nn.functional.one_hot(torch.arange(40), 64).to(BF) * 4)
        g = torch.Generator().manual_seed(2)
        key = torch.randn(dim, generator=g)
        q, k = w["l0.mix.q"], w["l0.mix.k"]
        for h in range(heads):
            q[h * dim:(h + 1) * dim, 1] = key.to(BF)                             # token 1 asks ...
        for h in range(kv_heads):
            k[h * dim:(h + 1) * dim, 0] = key.to(BF)                             # ... for token 0
        w["l0.mix.pb"].fill_(pb)
        w["l0.mix.v"][:, 0] *= 8
    m, w = build(raw, dtype, seed=1, edit=edit)
    return raw, m, w


@pytest.mark.parametrize("dim", [32, 64, 128, 160])
@DTYPES
def test_far_keys_in_prompts_and_decoding(dim, dtype):
    """The asked-for token at the edges of the kernels' key blocks, query blocks and context splits; its weight is ~1 where every other key's is
    ~0, so a key that is lost, doubled or displaced shows.  A planted mistake (the far token's key lost) in the reference is far outside the
    tolerance."""
    raw, m, w = far_model(dtype, dim)
    eng = m.step_engine(2, 1300)
    g = torch.Generator().manual_seed(0)
    base = torch.randint(2, 40, (1200,), generator=g).tolist()
    for n, places in ((130, (0, 1, 62, 63, 64, 65, 127, 128)), (700, (0, 63, 255, 256, 511, 512, 640)), (1200, (0, 127, 1023, 1024, 1150))):
        for far in places:
            toks = list(base[:n])
            toks[far], toks[n - 1] = 0, 1
            h = R.norm(R.embedding([toks[-1]], w["embed"].double(), w["pos"].double()), w["l0.norm1"].double(), raw["norm"]["eps"])
            ref = last_logits(raw, w, toks, h)
            lost = last_logits(raw, w, toks, h, drop=far)
            scale = float(ref.pow(2).mean().sqrt())
            assert float((ref - lost).pow(2).mean().sqrt()) / scale > 0.15, "the far key does not show"
            eng.launch([(0, 0, toks)])                                           # in the prompt
            p = eng.logits[0].double().cpu()
            eng.launch([(1, 0, toks[:-1])])                                      # decoded
            eng.launch([(1, n - 1, toks[-1:])])
            d = eng.logits[0].double().cpu()
            for got, what in ((p, "prompt"), (d, "decoded")):
                assert float((got - ref).pow(2).mean().sqrt()) / scale < TOL[dtype], (dim, n, far, what)


def last_logits(raw, w, toks, h_last, drop=None):
    """Reference logits of the last position only (one layer, attention alone); ``drop``: plant the mistake of losing that key."""
    w = {k: v.double() for k, v in w.items()}
    mix, eps, T = raw["layers"][0]["mixer"], raw["norm"]["eps"], len(toks)
    x = R.embedding(toks, w["embed"], w["pos"])
    h = R.norm(x, w["l0.norm1"], eps)
    H, G = mix["heads"], mix["kv_heads"]
    q = R.rms(R.linear(h[-1:], w["l0.mix.q"], w["l0.mix.q.b"]).view(H, -1), eps)
    k = R.rms(R.linear(h, w["l0.mix.k"], w["l0.mix.k.b"]).view(T, G, -1), eps)
    v = R.linear(h, w["l0.mix.v"], w["l0.mix.v.b"]).view(T, G, -1)
    dist = (T - 1 - torch.arange(T)).double()
    o = []
    for hd in range(H):
        g = hd // (H // G)
        a = torch.sigmoid(k[:, g] @ q[hd] * mix["scale"] - w["l0.mix.r1"][hd] * torch.log1p(w["l0.mix.r2"][hd] * dist) + w["l0.mix.pb"][hd])
        if drop is not None:
            a[drop] = 0
        o.append(a @ v[:, g])
    y = x[-1] + raw["residual_mult"] * R.linear(torch.cat(o)[None], w["l0.mix.o"], w["l0.mix.o.b"])[0]
    lg = R.linear(R.norm(y[None], w["final.norm"], eps), w["head"])[0]
    return raw["logit_softcap"] * torch.tanh(lg / raw["logit_softcap"])


@DTYPES
def test_old_state_shows_and_a_reset_does_not_leak(dtype):
    """Slow decay, a token with large step sizes at the start only: its trace in the state must reach a query hundreds of tokens later through every way of entering, and must
    be gone when the slot is handed to another request."""
    raw = raw_config([ssm(heads=2, groups=1, state=16, vdim=16, conv=4, norm_groups=1, ff=None)], width=48, vocab=40, max_positions=700)

    def edit(w):
        w["l0.mix.A_log"].fill_(-9.0)
        e0 = w["embed"][0].float()
        w["l0.mix.in"][-2:] = (0.2 * w["l0.mix.in"][-2:].float() + 6 * e0 / (e0.norm() * 48 ** 0.5)).to(BF)      # large step sizes for token 0
    m, w = build(raw, dtype, seed=4, edit=edit)
    toks = torch.randint(1, 40, (400,), generator=torch.Generator().manual_seed(3)).tolist()
    loud = [0] * 8 + toks[8:]
    ref_loud, ref = R.forward(raw, w, loud), R.forward(raw, w, toks)
    assert err(ref_loud[-20:], ref[-20:]) > 3 * TOL[dtype], "the early tokens do not show"
    eng = m.step_engine(1, 700)
    assert err(run(eng, 0, 0, loud), ref_loud) < TOL[dtype]
    assert err(run_cut(eng, 0, toks, [300, 64]), ref) < TOL[dtype]              # the same slot again
    assert err(run_cut(eng, 0, loud, [3, 100, 270]), ref_loud) < TOL[dtype]
    assert err(run_cut(eng, 0, toks[:30], []), ref[:30]) < TOL[dtype]


def test_long_decoding_stays_exact():
    """600 decoded tokens in fp32 and bf16 against whole prompts of the same kernels' fp32 form."""
    raw = dict(MODELS["looped"])
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
    m, toks, _ = zoo("looped", dtype)
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
    out = list(prompt)
    gaps = []
    for _ in range(n):
        lg = R.forward(raw, w, out)[-1]
        top = lg.topk(2)
        gaps.append(float(top.values[0] - top.values[1]))
        out.append(int(top.indices[0]))
    return out[len(prompt):], gaps


@pytest.mark.parametrize("chunk", [None, 5, 2])
def test_greedy_generation_through_the_scheduler(chunk):
    from onebit_amd.serving import ContinuousBatcher
    raw = raw_config([ssm(), att()], width=64, vocab=50, loop={"start": 0, "stop": 2, "times": 2}, cap=30.0)
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
    raw = raw_config([att(), ssm()], width=64, vocab=50)
    m, w = build(raw, F32, seed=2)
    ids = torch.tensor([tokens(7, 50, 1), tokens(7, 50, 2)])
    lg = m(ids.cuda())
    ref = torch.stack([R.forward(raw, w, r) for r in ids.tolist()])
    assert err(lg.view(14, -1), ref.view(14, -1)) < TOL[F32]
    out = m.generate(ids, 5)
    assert out.shape == (2, 12) and torch.equal(out[:, :7].cpu(), ids)
    for r, row in zip(ids.tolist(), out.tolist()):
        assert row[7] == int(R.forward(raw, w, r)[-1].argmax())
    eos = out[0, 8].item()
    cut = m.generate(ids[:1], 5, eos_token_id=eos)
    assert cut[0].tolist() == out[0, :9].tolist() or out[0, 7].item() == eos
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
    raw = raw_config([ssm(), att()], width=64, vocab=50, loop={"start": 1, "stop": 2, "times": 2})
    w = synthetic_weights(LebepelConfig.from_dict(raw), 6)
    (tmp_path / "config.json").write_text(json.dumps(raw))
    write_safetensors(str(tmp_path / "model.safetensors"), w)
    a, b = tokens(12, 50, 1), tokens(31, 50, 2)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:9], "want": [0, 8]}, {"id": "b", "tokens": b[:30], "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[9:10], "want": []}, {"id": "b", "tokens": b[30:], "want": [0]}], "end": ["b"]},
             {"step": 2, "entries": [{"id": "a", "tokens": a[10:11], "want": []}], "end": []},
             {"step": 3, "entries": [{"id": "a", "tokens": a[11:], "want": [0]}], "end": ["a"]},
             {"step": 4, "entries": [{"id": "c", "tokens": b[:5], "want": [4, ]}], "end": ["c"]}]
    ra, rb = R.forward(raw, w, a), R.forward(raw, w, b)
    for dtype, tol in (("bfloat16", TOL[BF]), ("float32", TOL[F32])):
        out = tmp_path / dtype
        assert trace_run(str(tmp_path), dtype, str(out), 64, lines=io.StringIO("\n".join(json.dumps(s) for s in steps))) == 0
        assert [l for l in capsys.readouterr().out.splitlines() if l.startswith("done")] == [f"done {i}" for i in range(5)]
        load = lambda i: torch.frombuffer(bytearray((out / f"{i}.f32").read_bytes()), dtype=torch.float32).view(-1, 50)
        assert err(load(0), ra[[0, 8]]) < tol and err(load(1), rb[[30]]) < tol and err(load(3), ra[[11]]) < tol and err(load(4), rb[[4]]) < tol
        assert not (out / "2.f32").exists()
    assert main(["generate", "--model", str(tmp_path), "--dtype", "float32", "--prompt", ",".join(map(str, a)), "--prompt", "3 4", "--max-new-tokens", "3"]) == 0
    rows = [json.loads(l) for l in capsys.readouterr().out.splitlines() if l.startswith("{")]
    assert len(rows) == 2 and rows[0]["tokens"][0] == int(ra[-1].argmax())


def test_launch_errors(zoo):
    m, toks, _ = zoo("plain", F32)
    eng = m.step_engine(2, 100)
    for items in ([(2, 0, [1])], [(0, 0, [1]), (0, 0, [2])], [(0, 98, [1, 2, 3])], [(0, 0, [61])], [(0, 0, [1, -1])], [(0, 0, [1, 2], [2])], []):
        with pytest.raises(ValueError):
            eng.launch(items)
    with pytest.raises(ValueError):
        m.step_engine(1, 5000)


def test_trace_runner_serves_the_other_family(tmp_path, capsys):
    """The same runner on a OneBit LLaMA folder: class, engine and precision chosen by config.json."""
    import io
    from onebit_amd.checkpoint import save_inference_checkpoint
    from onebit_amd.llama import OneBitLlamaConfig, build_synthetic_model
    from onebit_amd.trace import run as trace_run
    cfg = OneBitLlamaConfig(vocab_size=96, hidden_size=128, intermediate_size=352, num_hidden_layers=2, num_attention_heads=2, max_position_embeddings=64)
    model = build_synthetic_model(cfg, seed=1, device="cuda")
    save_inference_checkpoint(model, str(tmp_path))
    a, b = tokens(12, 96, 1), tokens(7, 96, 2)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:11], "want": [3, 10]}, {"id": "b", "tokens": b[:6], "want": [5]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[11:], "want": [0]}, {"id": "b", "tokens": b[6:], "want": []}], "end": ["a", "b"]}]
    assert trace_run(str(tmp_path), "bfloat16", str(tmp_path / "o"), 64, lines=io.StringIO("\n".join(map(json.dumps, steps)))) == 0
    capsys.readouterr()
    ra, rb = (model(torch.tensor([t], device="cuda"))[0].double().cpu() for t in (a, b))
    load = lambda i: torch.frombuffer(bytearray((tmp_path / "o" / f"{i}.f32").read_bytes()), dtype=torch.float32).view(-1, 96)
    assert err(load(0), torch.stack([ra[3], ra[10], rb[5]])) < 0.02 and err(load(1), ra[[11]]) < 0.02
