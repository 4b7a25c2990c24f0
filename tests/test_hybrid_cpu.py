"""Hybrid decoders on the host: packing, files, configuration, registry, slots, the plain restatement's own cross-checks, argument errors of
the native step (no GPU needed)."""
import ctypes
import io
import json

import pytest
import torch

from onebit_amd import _lib, registry
from onebit_amd.checkpoint import read_safetensors, write_safetensors
from onebit_amd.hybrid import _HLayer, _HModel, _HRun, _HSeg, _HState, k_tile, pack_fragments, unpack_fragments
from onebit_amd.lebepel import LebepelConfig, synthetic_weights
from onebit_amd.serving import Scheduler, SlotPool, cut_at_eos, eos_set
from oracle import lebepel_ref as R


def att(heads=4, kv_heads=2, dim=16, vdim=24, scale=0.3, ff=40):
    return {"type": "attention", "mixer": dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale), "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def ssm(heads=4, groups=2, state=16, vdim=8, conv=4, norm_groups=2, ff=40):
    return {"type": "mamba2", "mixer": dict(heads=heads, groups=groups, state=state, vdim=vdim, conv=conv, norm_groups=norm_groups),
            "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def raw_config(layers, width=40, vocab=61, loop=None, max_positions=96, mult=0.7, cap=9.0, eps=1e-4):
    c = {"architecture": "Lebepel", "layers": layers, "logit_softcap": cap, "max_positions": max_positions, "norm": {"eps": eps}, "residual_mult": mult,
         "vocab": vocab, "width": width}
    if loop is not None:
        c["loop"] = loop
    return c


@pytest.mark.parametrize("dtype", [torch.bfloat16, torch.float32])
def test_fragment_layout(dtype):
    kt = k_tile(dtype)
    w = torch.randn(37, 3 * kt - 5).to(dtype)
    p = pack_fragments(w, dtype)
    assert p.shape == (3, 3, 64, kt // 4) and p.is_contiguous()
    assert torch.equal(unpack_fragments(p, 37, w.shape[1]), w)
    for n, k in ((0, 0), (5, kt - 1), (36, 2 * kt + 3), (17, kt)):            # element (n, k): lane 16 (k % kt) // (kt / 4) + n % 16
        assert p[n // 16, k // kt, 16 * ((k % kt) // (kt // 4)) + n % 16, k % (kt // 4)] == w[n, k]
    assert float(unpack_fragments(p, 48, 3 * kt)[37:].abs().sum()) == 0 and float(unpack_fragments(p, 48, 3 * kt)[:, w.shape[1]:].abs().sum()) == 0


def test_safetensors_round_trip(tmp_path):
    t = {"a": torch.randn(3, 5).to(torch.bfloat16), "b.c": torch.arange(7, dtype=torch.int32), "e": torch.zeros(0, 4), "s": torch.tensor(2.5)}
    p = str(tmp_path / "x.safetensors")
    write_safetensors(p, t)
    back = read_safetensors(p)
    assert set(back) == set(t)
    for k in t:
        assert back[k].dtype == t[k].dtype and back[k].shape == t[k].shape and torch.equal(back[k], t[k])
    data = open(p, "rb").read()
    open(p, "wb").write(data[:-3])                                            # truncated data
    with pytest.raises(ValueError):
        read_safetensors(p)
    open(p, "wb").write(b"\xff" * 12)
    with pytest.raises(ValueError):
        read_safetensors(p)


def test_config_runs_and_errors():
    cfg = LebepelConfig.from_dict(raw_config([ssm(), att(), ssm(), att(ff=None)], loop={"start": 1, "stop": 3, "times": 3}))
    assert cfg.runs() == [(0, False), (1, False), (2, False), (1, True), (2, False), (1, True), (2, False), (3, False)] == R.layer_runs(cfg.to_dict())
    assert LebepelConfig.from_dict(cfg.to_dict()) == cfg
    assert LebepelConfig.from_dict(raw_config([att()])).runs() == [(0, False)]
    assert LebepelConfig.from_dict(raw_config([att(), att()], loop={"start": 0, "stop": 2, "times": 1})).runs() == [(0, False), (1, False)]
    s = cfg.tensor_shapes()
    assert s["l0.mix.in"] == (2 * 32 + 2 * 2 * 16 + 4, 40) and s["l1.mix.v"] == (48, 40) and "l3.mlp.up" not in s and s["l3.mix.o"] == (40, 96)
    for bad in (dict(raw_config([att()]), architecture="Other"), raw_config([dict(att(), type="window")]), raw_config([att(heads=3, kv_heads=2)]),
                raw_config([att()], loop={"start": 0, "stop": 2, "times": 2}), raw_config([dict(att(), mlp={"kind": "experts", "ff": 3})])):
        with pytest.raises(ValueError):
            LebepelConfig.from_dict(bad)


def test_registry_chooses_by_config(tmp_path):
    (tmp_path / "config.json").write_text(json.dumps(raw_config([att()])))
    assert registry.find_family(str(tmp_path)).name == "lebepel"
    (tmp_path / "config.json").write_text(json.dumps({"model_type": "bitllama", "vocab_size": 8}))
    fam = registry.find_family(str(tmp_path))
    assert fam.name == "bitllama" and not fam.float32
    (tmp_path / "config.json").write_text(json.dumps({"architecture": "Unknown"}))
    with pytest.raises(ValueError, match="no model family"):
        registry.find_family(str(tmp_path))


def test_trace_refuses_float32_without_kernels(tmp_path):
    from onebit_amd.trace import run
    (tmp_path / "config.json").write_text(json.dumps({"model_type": "bitllama"}))
    assert run(str(tmp_path), "float32", str(tmp_path / "out"), 8, lines=io.StringIO("")) == 3


def test_trace_session_slots():
    """Requests keep their slot and position, finished ones give theirs back, the engine grows when a batch needs more."""
    from onebit_amd.trace import TraceSession

    class Engine:
        def __init__(self):
            self.n_slots, self.seen = 2, []
            self.logits = torch.arange(400, dtype=torch.float32).view(100, 4)

        def grow(self, n):
            self.n_slots = n

        def launch(self, items):
            self.seen.append(items)

    class Fam:
        engine = staticmethod(lambda model, n, m: Engine())

    s = TraceSession(Fam, None, 32, n_slots=2)
    e = lambda i, t, w: {"id": i, "tokens": t, "want": w}
    out = s.step([e("a", [1, 2, 3], [2]), e("b", [4, 5], [0, 1])])
    assert out.shape == (3, 4) and s.engine.seen[-1] == [(0, 0, [1, 2, 3], [2]), (1, 0, [4, 5], [0, 1])]
    out = s.step([e("a", [7], []), e("b", [8], [0])], end=["a"])
    assert s.engine.seen[-1] == [(0, 3, [7]), (1, 2, [8])] and torch.equal(out, s.engine.logits[1:2])
    s.step([e("c", [1], [0]), e("d", [1, 1], [])])                             # a's slot again, one more than there are
    assert s.engine.n_slots == 4 and [it[:2] for it in s.engine.seen[-1]] == [(0, 0), (2, 0)]
    assert s.step([e("b", [2], [])], end=["b", "c", "d", "nobody"]) is None and len(s.pool) == 4


def test_slot_pool_and_scheduler():
    p = SlotPool(2)
    assert (p.take(), p.take(), len(p)) == (0, 1, 0)
    p.grow(4)
    assert p.take() == 2
    p.give(0)
    assert p.take() == 0 and p.take() == 3
    s = Scheduler(2, 16)
    s.add([1, 2], 1), s.add([3], 1), s.add([4], 1)
    items = s.plan()
    assert [it.req.slot for it in items] == [0, 1] and len(s.commit(items, [5, 6])) == 2
    assert [it.req.slot for it in s.plan()] == [1]                             # a freed slot is used again


def test_eos_rules():
    assert eos_set(None, 3, 2) == (None, 3) and eos_set(5, None, 1) == ({5}, 5)
    with pytest.raises(ValueError):
        eos_set(5, None, 2)
    assert cut_at_eos([[1, 5, 2], [1, 2, 3]], {5}, 0) == [[1, 5, 0], [1, 2, 3]] and cut_at_eos([[5, 1], [2, 5]], {5}, 9) == [[5, 9], [2, 5]]


# ---- the restatement against closed forms: what the GPU tests compare with must itself be right
def test_restatement_mechanisms():
    torch.manual_seed(0)
    x = torch.randn(5, 7, dtype=torch.float64)
    assert torch.allclose(R.rms(x, 0.25), x * (x.pow(2).mean(-1, keepdim=True) + 0.25).rsqrt())
    assert torch.allclose(R.norm(x, torch.zeros(7, dtype=torch.float64), 1e-6), R.rms(x, 1e-6))
    assert torch.allclose(R.silu(x), torch.nn.functional.silu(x)) and torch.allclose(R.softplus(x), torch.nn.functional.softplus(x))
    # convolution = torch's causal depthwise one
    taps, b = torch.randn(7, 3, dtype=torch.float64), torch.randn(7, dtype=torch.float64)
    ref = torch.nn.functional.conv1d(torch.nn.functional.pad(x.T[None], (2, 0)), taps[:, None], b, groups=7)[0].T
    assert torch.allclose(R.short_conv(x, taps, b), ref)
    # the recurrence, unrolled: y_t = sum_s exp(sum decays) dt_s (C_t . B_s) x_s + D x_t
    T, H, G, N, P = 6, 4, 2, 3, 2
    X, B, C = torch.randn(T, H, P, dtype=torch.float64), torch.randn(T, G, N, dtype=torch.float64), torch.randn(T, G, N, dtype=torch.float64)
    dt, A, D = torch.rand(T, H, dtype=torch.float64), torch.randn(H, dtype=torch.float64), torch.randn(H, dtype=torch.float64)
    y, S = R.ssm(X, B, C, dt, A, D)
    cum = torch.cumsum(-torch.exp(A) * dt, 0)
    for t in range(T):
        for h in range(H):
            e = D[h] * X[t, h] + sum(torch.exp(cum[t, h] - cum[s, h]) * dt[s, h] * (C[t, h // 2] @ B[s, h // 2]) * X[s, h] for s in range(t + 1))
            assert torch.allclose(y[t, h], e)
    # attention: one key -> sigmoid of its score, no normalisation; weights do not depend on other keys
    q, k, v = torch.randn(3, 4, 8, dtype=torch.float64), torch.randn(3, 2, 8, dtype=torch.float64), torch.randn(3, 2, 5, dtype=torch.float64)
    r1, r2, pb = torch.rand(4, dtype=torch.float64), torch.rand(4, dtype=torch.float64), torch.randn(4, dtype=torch.float64)
    o = R.sigmoid_attention(q, k, v, 0.7, r1, r2, pb, 1e-5)
    un = lambda z: z / (z.pow(2).mean() + 1e-5).sqrt()
    assert torch.allclose(o[0, 3], torch.sigmoid(0.7 * un(q[0, 3]) @ un(k[0, 1]) + pb[3]) * v[0, 1])
    e = sum(torch.sigmoid(0.7 * un(q[2, 1]) @ un(k[j, 0]) - r1[1] * torch.log(1 + r2[1] * (2 - j)) + pb[1]) * v[j, 0] for j in range(3))
    assert torch.allclose(o[2, 1], e)
    g = R.gated_group_norm(x[:, :6], x[:, 1:], torch.ones(6, dtype=torch.float64), 3, 0.0)
    assert torch.allclose(g.view(5, 3, 2).pow(2).mean(-1), torch.ones(5, 3, dtype=torch.float64))


def test_restatement_is_causal_and_loops():
    cfg = raw_config([ssm(), att()], loop={"start": 0, "stop": 2, "times": 2})
    w = synthetic_weights(LebepelConfig.from_dict(cfg), seed=3)
    toks = [7, 1, 60, 22, 22, 5]
    col = []
    full = R.forward(cfg, w, toks, collect=col)
    assert torch.allclose(R.forward(cfg, w, toks[:4]), full[:4]) and len(col) == 4
    flat = R.forward(dict(cfg, loop=None), w, toks, collect=(c2 := []))
    assert torch.allclose(col[1], c2[1]) and not torch.allclose(full, flat)
    assert float(full.abs().max()) < cfg["logit_softcap"]


# ---- the native step refuses bad arguments before it launches anything
def _fake_model(a, **kw):
    L = (_HLayer * 1)()
    l = L[0]
    l.kind, l.nt_mix, l.nt_aux, l.nt_in, l.mix_k, l.act_k = 0, 8, 0, 12, 96, 32
    l.w_in = l.w_out = l.norm_w = a
    l.heads, l.vdim, l.kv_heads, l.dim, l.kp, l.vp, l.unit_rms, l.scale = 4, 24, 2, 8, 64, 64, 1, 0.5
    for k, v in kw.pop("layer", {}).items():
        setattr(l, k, v)
    runs = (_HRun * 1)(_HRun(0, 0, a, a))
    m = _HModel(ctypes.sizeof(_HModel), _lib.HYB_BF16, 40, 64, 61, 1, 1, 3, 32, 32, 1e-5, 1.0, 0.5, 0.0, a, a, a, a, L, runs)
    for k, v in kw.items():
        setattr(m, k, v)
    return m, (L, runs)


def test_native_step_rejects_bad_arguments():
    lib = _lib.load_hybrid()
    E_ARG, E_SHAPE, E_DTYPE, E_WSPACE = -1, -2, -4, -5
    buf = ctypes.create_string_buffer(4096)
    a = (ctypes.addressof(buf) + 255) & ~255
    m, keep = _fake_model(a)
    size = lambda mm, rows=8, outs=8, dec=3, sp=4: lib.onebit_hybrid_workspace_bytes(ctypes.byref(mm), rows, outs, dec, sp)
    assert size(m) > 0 and size(m, rows=1000) > size(m) and size(m, rows=0) == 0
    for kw, layer in ((dict(struct_size=8), {}), (dict(width_pad=48), {}), (dict(dtype=7), {}), (dict(max_len=64), {}), ({}, dict(kind=5)), ({}, dict(nt_in=11)),
                      ({}, dict(kv_heads=3)), ({}, dict(mix_k=64)), ({}, dict(act_k=0)), ({}, dict(nt_mix=4)), ({}, dict(kind=1))):
        bad, k2 = _fake_model(a, layer=layer, **kw)
        assert size(bad) == 0, (kw, layer)
    seg = (_HSeg * 1)(_HSeg(1, 4, 0, 0))
    def step(mm=m, rows=5, outs=8, **kw):
        st = _HState(ctypes.sizeof(_HState), 5, 1, 1, 1, 0, 128, 1, a, a, a, a, seg, a, a, a, None, a, 1 << 40)
        for k, v in kw.items():
            setattr(st, k, v)
        return lib.onebit_hybrid_step(ctypes.byref(mm), ctypes.byref(st), rows, outs, 3, 4, None)
    assert step(struct_size=4) == E_ARG and b"struct_size" in lib.onebit_hybrid_last_error()
    assert step(n_rows=6) == E_SHAPE and step(rows=4) == E_SHAPE and step(attn_chunk=96) == E_SHAPE and step(attn_splits=5) == E_SHAPE
    assert step(n_rows=7, rows=9) == E_SHAPE and b"n_rows" in lib.onebit_hybrid_last_error()
    assert step(workspace_bytes=64) == E_WSPACE and step(logits=None) == E_ARG and step(n_rows=0, n_dec=0, n_seg=0) == 0
    seg[0].slot = 3
    assert step() == E_SHAPE and b"segment 0" in lib.onebit_hybrid_last_error()
    seg[0].slot, seg[0].past = 0, 30
    assert step() == E_SHAPE
    assert lib.onebit_hybrid_gemm(a, a, a, 9, 1, 1, 1, 1, None) == E_DTYPE and lib.onebit_hybrid_gemm(a, a, a, 2, 1, 3, 1, 2, None) == E_ARG
    assert lib.onebit_hybrid_gemm_splits(256, 472, 1) >= 1
    with pytest.raises(ValueError):
        _lib.check_hybrid(E_SHAPE, "x")


def test_header_symbols_are_bound():
    import os
    import re
    text = open(os.path.join(os.path.dirname(os.path.dirname(os.path.abspath(__file__))), "include", "onebit_hybrid.h")).read()
    assert set(re.findall(r"\b(onebit_hybrid_\w+)\s*\(", text)) == set(_lib.HYBRID_SYMBOLS)


def test_cli_arguments(capsys):
    from onebit_amd.cli import main, trace_main
    with pytest.raises(SystemExit):
        trace_main(["--model", "x"])
    with pytest.raises(SystemExit):
        main(["generate"])
    with pytest.raises(SystemExit) as e:
        main(["--help"])
    assert e.value.code == 0 and "generate" in capsys.readouterr().out
