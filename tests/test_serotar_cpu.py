"""Serotar on the host: configuration, registry, tensors, packing, the order of a step's rows, the plain restatement's own cross-checks, argument
errors of the native step (no GPU needed)."""
import ctypes
import json

import pytest
import torch

from onebit_amd import _lib, registry
from onebit_amd.hybrid import (ExpertMixture, GatedFeedForward, HybridLayer, LatentAttention, TokenInput, XieluFeedForward, _HLayer, _HModel, _HRun, _HSeg, _HState, _Packed,
                               unpack_fragments)
from onebit_amd.serotar import SerotarConfig, SerotarForCausalLM, synthetic_weights
from oracle import serotar_ref as R


def dense(ff=40):
    return {"kind": "dense", "ff": ff}


def moe(experts=6, top=2, identity=2, groups=(4, 2), ff=24, shared=32):
    r = {"experts": experts, "top": top}
    if identity:
        r["identity"] = identity
    if groups:
        r["groups"] = {"count": groups[0], "keep": groups[1]}
    m = {"kind": "moe", "expert": {"ff": ff}, "router": r}
    if shared:
        m["shared"] = {"ff": shared}
    return m


def layer(mlp=None, heads=3, dim=16, vdim=24, q_rank=20, kv_rank=36, scale=0.3):
    return {"type": "latent_attention", "mixer": dict(heads=heads, dim=dim, vdim=vdim, q_rank=q_rank, kv_rank=kv_rank, scale=scale), "mlp": mlp}


def raw_config(layers, width=52, vocab=61, scale=1.5, bigram=(97, 13, 5), side=10, eps=1e-4):
    c = {"architecture": "Serotar", "embedding": {"scale": scale}, "layers": layers, "norm": {"eps": eps}, "vocab": vocab, "width": width}
    if bigram:
        c["embedding"]["bigram"] = dict(zip(("buckets", "mul_prev", "mul_cur"), bigram))
    if side:
        c["token_side"] = {"dim": side}
    return c


def test_config_and_tensors():
    cfg = SerotarConfig.from_dict(raw_config([layer(dense()), layer(moe()), layer(None)]))
    assert SerotarConfig.from_dict(cfg.to_dict()) == cfg
    s = cfg.tensor_shapes()
    assert s["bigram"] == (98, 52) and s["side.embed"] == (61, 30) and s["l1.mlp.router"] == (8, 52) and s["l1.mlp.e5.down"] == (52, 24)
    assert s["l0.mlp.act"] == (2,) and s["l2.dwa"] == (4,) and "l2.norm2" not in s and "l2.ls2" not in s and s["l0.norm1"] == () and s["final.norm"] == ()
    assert s["l1.mix.uq"] == (48, 20) and s["l1.mix.uv"] == (72, 36) and s["l1.mix.o"] == (52, 72) and "l1.mlp.e6.down" not in s
    plain = SerotarConfig.from_dict(raw_config([layer(moe(identity=0, groups=None, shared=0))], bigram=None, side=0)).tensor_shapes()
    assert not {"bigram", "side.embed", "l0.side.gate", "l0.mlp.shared.up"} & set(plain) and plain["l0.mlp.correction"] == (6,)
    for bad in (dict(raw_config([layer()]), architecture="Other"), raw_config([dict(layer(), type="attention")]), raw_config([layer({"kind": "gated", "ff": 3})]),
                raw_config([layer(moe(groups=(3, 1)))]), raw_config([layer(moe(top=5, groups=(4, 2)))]), raw_config([layer(moe(groups=(4, 5)))])):
        with pytest.raises(ValueError):
            SerotarConfig.from_dict(bad)
    w = synthetic_weights(cfg, 0)
    del w["l1.mlp.e3.up"]
    with pytest.raises(ValueError, match="l1.mlp.e3.up"):
        SerotarForCausalLM(cfg, w, device="cpu")
    w = synthetic_weights(cfg, 0)
    w["l0.mix.uk"] = w["l0.mix.uk"][:5]
    with pytest.raises(ValueError, match="l0.mix.uk"):
        SerotarForCausalLM(cfg, w, device="cpu")


def test_registry_chooses_by_config(tmp_path):
    (tmp_path / "config.json").write_text(json.dumps(raw_config([layer()])))
    fam = registry.find_family(str(tmp_path))
    assert fam.name == "serotar" and fam.float32 and fam.serving_dtype == torch.bfloat16


@pytest.mark.parametrize("dtype", [torch.bfloat16, torch.float32])
def test_packing_of_latent_attention_and_experts(dtype):
    cfg = SerotarConfig.from_dict(raw_config([layer(moe(), dim=72, vdim=40)]))
    w = synthetic_weights(cfg, 1, torch.float32)
    W, H, m = 52, 3, cfg.layers[0]["mixer"]
    att = LatentAttention(H, 72, 40, 0.3, *[w["l0.mix." + n] for n in ("dq", "dq.norm", "uq", "dkv", "dkv.norm", "uk", "uv", "o")])
    g = lambda p: GatedFeedForward(w[p + "gate"], w[p + "up"], w[p + "down"])
    mix = ExpertMixture([g(f"l0.mlp.e{e}.") for e in range(6)], w["l0.mlp.router"], w["l0.mlp.correction"], 2, 2, 4, 2, g("l0.mlp.shared."))
    p = _Packed(HybridLayer(None, att, mix, sequential=True), W, 64, dtype)
    c, l = p.c, p.c.latent
    bf = dtype == torch.bfloat16
    assert (l.tiled, l.flash, l.rp, c.kp, l.vdp) == ((1, 1, 64, 128, 64) if bf else (0, 0, 64, 96, 64))
    by = {t.data_ptr(): t for t in p.keep}
    r = lambda t: t.to(dtype).float()
    uk = unpack_fragments(by[l.w_uk], H * l.rp, c.kp).float().view(H, l.rp, c.kp)            # transposed per head, padding zero
    assert torch.equal(uk[:, :36, :72], r(w["l0.mix.uk"]).view(H, 72, 36).transpose(1, 2)) and float(uk[:, 36:].abs().sum() + uk[:, :, 72:].abs().sum()) == 0
    uv = unpack_fragments(by[l.w_uv], H * l.vdp, l.rp).float().view(H, l.vdp, l.rp)
    assert torch.equal(uv[:, :40, :36], r(w["l0.mix.uv"]).view(H, 40, 36)) and float(uv[:, 40:].abs().sum()) == 0
    o = unpack_fragments(by[c.w_out], W, H * l.vdp).float().view(W, H, l.vdp)
    assert torch.equal(o[:, :, :40], r(w["l0.mix.o"]).view(W, H, 40)) and float(o[:, :, 40:].abs().sum()) == 0
    f = c.ff
    assert (f.experts, f.identity, f.nt_aux, f.nt_expert, f.nt_gated) == (6, 2, 2, 4, 4)
    e_in = by[f.w_expert_in].view(6, f.nt_expert, -1, 64, by[f.w_expert_in].shape[-1])
    one = unpack_fragments(e_in[4], 64, W).float().view(2, 2, 16, W)                          # 16 gate rows, 16 up rows, ...
    assert torch.equal(one[:, 0].reshape(32, W)[:24], r(w["l0.mlp.e4.gate"])) and torch.equal(one[:, 1].reshape(32, W)[:24], r(w["l0.mlp.e4.up"]))
    e_out = by[f.w_expert_out].view(6, 4, -1, 64, by[f.w_expert_out].shape[-1])
    assert torch.equal(unpack_fragments(e_out[2], W, 24).float(), r(w["l0.mlp.e2.down"]))
    router = unpack_fragments(by[f.w_gated_in], 8, W).float()
    assert torch.equal(router, r(w["l0.mlp.router"]))
    if bf:
        kv = unpack_fragments(by[l.w_kv], 2 * H * 128, 36).float().view(2, H, 128, 36)
        assert torch.equal(kv[0, :, :72], r(w["l0.mix.uk"]).view(H, 72, 36)) and torch.equal(kv[1, :, :40], r(w["l0.mix.uv"]).view(H, 40, 36))
        assert float(kv[0, :, 72:].abs().sum() + kv[1, :, 40:].abs().sum()) == 0


def test_parts_that_do_not_go_together():
    t = torch.zeros
    att = LatentAttention(1, 4, 4, 1.0, t(4, 8), t(4), t(4, 4), t(4, 8), t(4), t(4, 4), t(4, 4), t(8, 4))
    xi = XieluFeedForward(t(4, 8), t(8, 4), 0.0, 0.0)
    for lay in (HybridLayer(t(8), att, None), HybridLayer(t(8), att, xi), HybridLayer(None, att, None, sequential=False),
                HybridLayer(None, att, None, sequential=True, token_input=TokenInput(t(4, 8), t(8, 4), t(8), 2)),
                HybridLayer(None, att, ExpertMixture([GatedFeedForward(t(4, 8), t(4, 8), t(8, 4))], t(3, 8), t(3), 1, 1), sequential=True)):
        with pytest.raises(ValueError):
            _Packed(lay, 8, 32, torch.bfloat16, t(5, 4))


# ---- the restatement against closed forms
def test_restatement_mechanisms():
    torch.manual_seed(0)
    x = torch.randn(5, 7, dtype=torch.float64)
    assert torch.allclose(R.gelu_tanh(x), torch.nn.functional.gelu(x, approximate="tanh"))
    assert torch.allclose(R.silu(x), torch.nn.functional.silu(x)) and torch.allclose(R.softplus(x), torch.nn.functional.softplus(x))
    p, q = torch.tensor(0.3, dtype=torch.float64), torch.tensor(-1.2, dtype=torch.float64)
    z = torch.tensor([2.0, -2.0, 0.0, 1e-9, -1e-9], dtype=torch.float64)
    sp = lambda v: float(torch.nn.functional.softplus(v))
    y = R.xielu(z, p, q)
    assert abs(float(y[0]) - (4 * sp(p) + 1)) < 1e-12 and abs(float(y[1]) - ((0.5 + sp(q)) * (2.718281828459045 ** -2 + 1) - 1)) < 1e-12 and float(y[2]) == 0
    assert abs(float(y[3]) / 1e-9 - 0.5) < 1e-6 and abs(float(y[4]) / -1e-9 - 0.5) < 1e-6      # slope 1/2 from both sides
    qh, k, v = torch.randn(6, 2, 8, dtype=torch.float64), torch.randn(6, 2, 8, dtype=torch.float64), torch.randn(6, 2, 5, dtype=torch.float64)
    ref = torch.nn.functional.scaled_dot_product_attention(qh.transpose(0, 1), k.transpose(0, 1), v.transpose(0, 1), is_causal=True, scale=0.7).transpose(0, 1)
    assert torch.allclose(R.softmax_attention(qh, k, v, 0.7), ref)
    assert R.bigram_rows([4, 9, 9], dict(buckets=10, mul_prev=3, mul_cur=7)) == [10, (12 + 63) % 10, (27 + 63) % 10]


def test_restatement_routing():
    s = torch.tensor([0.4, 0.1, 0.05, 0.25, 0.15, 0.05], dtype=torch.float64)
    zero = torch.zeros(6, dtype=torch.float64)
    assert R.choose(s, zero, dict(top=2)) == [0, 3]
    assert R.choose(s, torch.tensor([-1., 0, 0, 0, 0, 0.3], dtype=torch.float64), dict(top=2)) == [5, 3]
    # groups {0 1} {2 3} {4 5}, best one by its largest member; the others are out even when every choice score is negative
    assert R.choose(s, zero, dict(top=2, groups=dict(count=3, keep=1))) == [0, 1]
    assert R.choose(s, zero - 1, dict(top=4, groups=dict(count=3, keep=2))) == [0, 3, 1, 2]
    # weights are the plain scores, not renormalised; identity experts return their input; the shared expert is added
    h = torch.randn(2, 4, dtype=torch.float64)
    w = {"p.router": torch.randn(3, 4, dtype=torch.float64), "p.correction": torch.tensor([0., 0., 9.], dtype=torch.float64)}
    for e in ("e0", "e1", "shared"):
        w.update({f"p.{e}.gate": torch.randn(5, 4, dtype=torch.float64), f"p.{e}.up": torch.randn(5, 4, dtype=torch.float64), f"p.{e}.down": torch.randn(4, 5, dtype=torch.float64)})
    out = R.mixture(h, w, "p.", {"router": dict(experts=2, identity=1, top=1), "shared": {"ff": 5}})
    s = torch.softmax(h @ w["p.router"].T, -1)
    assert torch.allclose(out, s[:, 2:] * h + R.expert(h, w, "p.shared."))


def test_restatement_is_causal_and_depends_on_every_part():
    cfg = raw_config([layer(dense()), layer(moe()), layer(None)])
    w = synthetic_weights(SerotarConfig.from_dict(cfg), 3)
    toks = [7, 1, 60, 22, 22, 5]
    col = []
    full = R.forward(cfg, w, toks, collect=col)
    assert torch.allclose(R.forward(cfg, w, toks[:4]), full[:4]) and len(col) == 3
    base = float(full.norm())
    for name in sorted(w):
        if ".mlp.e" in name:
            continue                                                          # (not every expert is used)
        w2 = dict(w)
        w2[name] = w[name].float() + (torch.randn(w[name].shape) if w[name].dim() else 0.5)       # (one weight for all columns: not the same direction)
        assert float((R.forward(cfg, w2, toks) - full).norm()) > 1e-3 * base, name


# ---- order of a step's rows: single tokens, short chunks, long chunks
def test_stage_puts_short_chunks_first(monkeypatch):
    from onebit_amd.engine import ItemStage
    monkeypatch.setattr(torch.Tensor, "pin_memory", lambda self: self)
    monkeypatch.setattr(torch.cuda, "Event", lambda: type("E", (), {"record": lambda self, s: None, "synchronize": lambda self: None})())
    monkeypatch.setattr(torch.cuda, "current_stream", lambda d=None: None)
    st = ItemStage(torch.device("cpu"), 6, 100, 50, short=4)
    st.ensure(64)
    g = st.stage([(0, 0, [1] * 9), (1, 30, [2] * 3, [0, 2]), (2, 7, [3]), (3, 50, [4] * 4), (4, 0, [5] * 20)])
    assert g.segs == [(1, 3, 1, 30), (4, 4, 3, 50), (8, 9, 0, 0), (17, 20, 4, 0)] and (g.n_dec, g.n_short, g.n_rows, g.dec_ctx) == (1, 2, 37, 54)
    rows = st._np[0]
    assert rows[:8].tolist() == [3, 2, 2, 2, 4, 4, 4, 4] and rows[4 * 64:4 * 64 + 6].tolist() == [16, 1, 3, 0, 7, 36]
    g = ItemStage.stage(st, [(0, 0, [1] * 2)])
    assert (g.n_dec, g.n_short, g.dec_ctx) == (0, 1, 2)


# ---- the native step refuses bad arguments before it launches anything
def _fake_model(a, latent={}, ff={}, side={}, layer={}, **kw):
    L = (_HLayer * 1)()
    l = L[0]
    l.kind, l.form, l.nt_mix, l.nt_in, l.mix_k = 2, 1, 6, 6, 128
    l.w_in = l.w_out = a
    l.heads, l.dim, l.vdim, l.kp, l.vp, l.scale = 2, 24, 40, 64, 64, 0.5
    d = dict(q_rank=30, kv_rank=60, nt_q=2, rp=64, tiled=1, flash=64, vdp=64, qn_w=a, kvn_w=a, w_uq=a, w_uk=a, w_uv=a, w_kv=a)
    for k, v in dict(d, **latent).items():
        setattr(l.latent, k, v)
    d = dict(nt_gated=4, nt_aux=2, nt_expert=4, experts=6, identity=2, top=2, groups=4, keep=2, w_gated_in=a, w_gated_out=a, w_expert_in=a, w_expert_out=a, correction=a)
    for k, v in dict(d, **ff).items():
        setattr(l.ff, k, v)
    for k, v in dict(dict(dim=10, nt=2, w_gate=a, w_proj=a, norm_w=a, table=a), **side).items():
        setattr(l.side, k, v)
    for k, v in layer.items():
        setattr(l, k, v)
    runs = (_HRun * 1)(_HRun(0, 0, a, None))
    m = _HModel(ctypes.sizeof(_HModel), _lib.HYB_BF16, 40, 64, 61, 1, 1, 3, 40, 1 << 20, 1e-5, 0.0, 1.0, 0.0, a, None, a, a, L, runs, 1.0, a, 97, 3, 5, a, 10)
    for k, v in kw.items():
        setattr(m, k, v)
    return m, (L, runs)


def test_native_step_rejects_bad_arguments():
    lib = _lib.load_hybrid()
    buf = ctypes.create_string_buffer(4096)
    a = (ctypes.addressof(buf) + 255) & ~255
    size = lambda mm, rows=8, outs=8, dec=3, sp=4: lib.onebit_hybrid_workspace_bytes(ctypes.byref(mm), rows, outs, dec, sp)
    m, keep = _fake_model(a)
    assert size(m) > 0 and size(m, rows=4000) > size(m)
    for kw in (dict(latent=dict(rp=96)), dict(latent=dict(rp=32)), dict(latent=dict(nt_q=1)), dict(latent=dict(vdp=32)), dict(latent=dict(w_uk=None)), dict(latent=dict(w_kv=None)),
               dict(latent=dict(tiled=0)), dict(ff=dict(nt_gated=2)), dict(ff=dict(nt_expert=2)), dict(ff=dict(groups=3)), dict(ff=dict(keep=5)), dict(ff=dict(top=5)), dict(ff=dict(experts=0)),
               dict(ff=dict(nt_plain=2, w_plain_in=a, w_plain_out=a)), dict(ff=dict(correction=None)), dict(ff=dict(experts=400, identity=0, groups=1, keep=1)), dict(side=dict(nt=1)),
               dict(side=dict(dim=40)), dict(side=dict(table=None)), dict(side_cols=4), dict(layer=dict(form=0)), dict(layer=dict(form=3)), dict(layer=dict(act_k=32)), dict(layer=dict(mix_k=64)),
               dict(layer=dict(kp=96)), dict(layer=dict(b_in=a)), dict(token_history=None), dict(buckets=0), dict(dtype=_lib.HYB_F32)):
        bad, k2 = _fake_model(a, **kw)
        assert size(bad) == 0, kw
    f32, k3 = _fake_model(a, latent=dict(tiled=0, flash=0), dtype=_lib.HYB_F32)
    assert size(f32) > 0
    segs = (_HSeg * 2)(_HSeg(1, 4, 0, 0), _HSeg(5, 17, 1, 3))
    def step(mm=m, **kw):
        st = _HState(ctypes.sizeof(_HState), 22, 1, 2, 1, 1, 128, 1, a, a, a, a, segs, a, a, a, None, a, 64)
        for k, v in kw.items():
            setattr(st, k, v)
        return lib.onebit_hybrid_step(ctypes.byref(mm), ctypes.byref(st), 22, 8, 3, 4, None)
    assert step() == -5                                                        # everything in order but the workspace
    assert step(n_short=2) == -2 and b"short" in lib.onebit_hybrid_last_error()
    assert step(n_short=3) == -1 and step(n_short=-1) == -1 and step(attn_chunk=64) == -2
    segs[0].past = 126                                                         # beyond what the decode attention is asked to cover, and beyond the cache
    assert step() == -2
