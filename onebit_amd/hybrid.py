"""Hybrid decoders: dense-weight decoder-only models whose layers mix different sequence mixers, on ``libonebit_hybrid.so``
(include/onebit_hybrid.h).

A design describes itself with the parts below -- ``SigmoidAttention`` / ``StateSpace`` mixers, ``GatedFeedForward``, ``HybridLayer``,
the order of layer runs -- and inherits packing, cache / state, the step engine, generation and evaluation from ``HybridDecoder``.
Every layer is the parallel form  x += mult * (mixer(norm(x)) + ff(norm(x)))  as two matrix products: mixer and feed-forward read one
normalised row, so their input projections are ONE weight matrix, and their output projections act on disjoint column ranges of one
row, so they are one matrix too (csrc/ob_dense.h has the packed layout).

``StateSlots`` holds what requests leave between steps, per layer RUN (a layer that a loop repeats has an entry for each repetition): keys and
values, or the fp32 recurrent state and the ring of convolution inputs.  ``HybridStep`` is the step engine with ``MixedStep``'s
interface: items in, greedy tokens and logits out; single-token steps replay a HIP graph."""
from __future__ import annotations

import ctypes
from dataclasses import dataclass
from typing import Dict, List, Optional, Sequence, Tuple

import torch
import torch.nn.functional as F

from . import _lib
from .engine import ItemStage

_vp, _i32, _f, _u64 = ctypes.c_void_p, ctypes.c_int32, ctypes.c_float, ctypes.c_uint64


class _HLayer(ctypes.Structure):
    _fields_ = [("kind", _i32), ("nt_mix", _i32), ("nt_aux", _i32), ("nt_in", _i32), ("mix_k", _i32), ("act_k", _i32),
                ("w_in", _vp), ("w_out", _vp), ("b_in", _vp), ("b_out", _vp), ("norm_w", _vp), ("heads", _i32), ("vdim", _i32),
                ("kv_heads", _i32), ("dim", _i32), ("kp", _i32), ("vp", _i32), ("unit_rms", _i32), ("scale", _f),
                ("r1", _vp), ("r2", _vp), ("pb", _vp),
                ("groups", _i32), ("state", _i32), ("taps", _i32), ("norm_groups", _i32), ("sp", _i32),
                ("conv_w", _vp), ("conv_b", _vp), ("dt_bias", _vp), ("A_log", _vp), ("D", _vp), ("gnorm_w", _vp)]


class _HRun(ctypes.Structure):
    _fields_ = [("layer", _i32), ("add_embedding", _i32), ("s0", _vp), ("s1", _vp)]


class _HModel(ctypes.Structure):
    _fields_ = [("struct_size", _u64), ("dtype", _i32), ("width", _i32), ("width_pad", _i32), ("vocab", _i32), ("n_layers", _i32),
                ("n_runs", _i32), ("n_slots", _i32), ("max_len", _i32), ("max_pos", _i32), ("eps", _f), ("norm_off", _f), ("mult", _f),
                ("softcap", _f), ("embed", _vp), ("pos_embed", _vp), ("final_norm", _vp), ("head", _vp),
                ("layers", ctypes.POINTER(_HLayer)), ("runs", ctypes.POINTER(_HRun))]


class _HSeg(ctypes.Structure):
    _fields_ = [("row0", _i32), ("n", _i32), ("slot", _i32), ("past", _i32)]


class _HState(ctypes.Structure):
    _fields_ = [("struct_size", _u64), ("n_rows", _i32), ("n_dec", _i32), ("n_seg", _i32), ("n_out", _i32), ("attn_chunk", _i32),
                ("attn_splits", _i32), ("tokens", _vp), ("row_slot", _vp), ("row_pos", _vp), ("row_off", _vp),
                ("segs", ctypes.POINTER(_HSeg)), ("out_rows", _vp), ("logits", _vp), ("next_tokens", _vp), ("residuals", _vp),
                ("workspace", _vp), ("workspace_bytes", ctypes.c_size_t)]


# ---------------------------------------------------------------------------------------------------------- packed weights --
def _up(n: int, m: int) -> int:
    return -(-n // m) * m


def k_tile(dtype: torch.dtype) -> int:
    """Columns of one 16-row tile of the fragment-major layout (64 bytes of a row)."""
    return 64 // torch.empty(0, dtype=dtype).element_size()


def pack_fragments(w: torch.Tensor, dtype: torch.dtype, k_pad: Optional[int] = None) -> torch.Tensor:
    """[N, K] -> fragment-major [ceil(N / 16), K_pad / KT, 64, KT / 4]: lane l of a tile holds row l % 16, columns (l // 16) KT / 4 .. ;
    rows and columns beyond N and K are zero."""
    N, K = w.shape
    kt = k_tile(dtype)
    kp = _up(K, kt) if k_pad is None else k_pad
    t = torch.zeros(_up(N, 16), kp, dtype=dtype, device=w.device)
    t[:N, :K] = w
    return t.view(-1, 16, kp // kt, 4, kt // 4).permute(0, 2, 3, 1, 4).contiguous().view(-1, kp // kt, 64, kt // 4)


def unpack_fragments(p: torch.Tensor, N: int, K: int) -> torch.Tensor:
    """The inverse of ``pack_fragments``."""
    n16, nkt, _, e = p.shape
    return p.view(n16, nkt, 4, 16, e).permute(0, 3, 1, 2, 4).reshape(n16 * 16, nkt * 4 * e)[:N, :K]


def _pad_rows(w: torch.Tensor, n: int) -> torch.Tensor:
    return F.pad(w, (0, 0, 0, n - w.shape[0]))


# --------------------------------------------------------------------------------------------------------- layer descriptions --
@dataclass
class SigmoidAttention:
    """Attention with unnormalised sigmoid weights: w = sigmoid(q.k scale - r1 ln(1 + r2 distance) + pb); ``unit_rms``: queries and keys
    divided by their root mean square per head.  ``r1`` / ``r2`` (together) and ``pb`` [heads] may be None."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    q: torch.Tensor
    k: torch.Tensor
    v: torch.Tensor
    o: torch.Tensor
    q_bias: Optional[torch.Tensor] = None
    k_bias: Optional[torch.Tensor] = None
    v_bias: Optional[torch.Tensor] = None
    o_bias: Optional[torch.Tensor] = None
    unit_rms: bool = True
    r1: Optional[torch.Tensor] = None
    r2: Optional[torch.Tensor] = None
    pb: Optional[torch.Tensor] = None


@dataclass
class StateSpace:
    """Scalar-decay state-space mixer: ``w_in`` rows [z | x | B | C | dt], a causal convolution over x | B | C, state ``state`` x ``vdim``
    per head, gate silu(z) before a norm over ``norm_groups`` equal parts."""
    heads: int
    groups: int
    state: int
    vdim: int
    norm_groups: int
    w_in: torch.Tensor
    conv_w: torch.Tensor          # [channels, taps]
    conv_b: torch.Tensor
    dt_bias: torch.Tensor
    A_log: torch.Tensor
    D: torch.Tensor
    norm: torch.Tensor
    o: torch.Tensor


@dataclass
class GatedFeedForward:
    """down(silu(gate h) * up h)."""
    gate: torch.Tensor
    up: torch.Tensor
    down: torch.Tensor


@dataclass
class HybridLayer:
    norm: torch.Tensor
    mixer: object
    mlp: Optional[GatedFeedForward]


class _Packed:
    """A layer on the device: the two fragment-major matrices and everything else as fp32 vectors, behind a filled ``_HLayer``."""

    def __init__(self, layer: HybridLayer, width: int, width_pad: int, dtype: torch.dtype):
        kt, m, mlp = k_tile(dtype), layer.mixer, layer.mlp
        self.keep: List[torch.Tensor] = []

        def f32(t):
            if t is None:
                return None
            t = t.detach().float().contiguous()
            self.keep.append(t)
            return t.data_ptr()

        c = self.c = _HLayer()
        att = isinstance(m, SigmoidAttention)
        if att:
            plain, aux = torch.cat([m.q, m.k, m.v]), None
            bias = None
            if any(b is not None for b in (m.q_bias, m.k_bias, m.v_bias)):
                bias = torch.cat([torch.zeros(w.shape[0], device=w.device) if b is None else b.float()
                                  for w, b in ((m.q, m.q_bias), (m.k, m.k_bias), (m.v, m.v_bias))])
        else:
            plain, aux, bias = m.w_in[:-m.heads], m.w_in[-m.heads:], None
        nt_mix, nt_aux = -(-plain.shape[0] // 16), 0 if aux is None else -(-aux.shape[0] // 16)
        nt_mix += (nt_mix + nt_aux) & 1                                  # gate / up tile pairs start at an even tile
        rows = [_pad_rows(plain, 16 * nt_mix)] + ([] if aux is None else [_pad_rows(aux, 16 * nt_aux)])
        ff_tiles = 0
        if mlp is not None:
            ff_tiles = -(-mlp.gate.shape[0] // 16)
            g, u = (_pad_rows(t, 16 * ff_tiles).view(ff_tiles, 16, width) for t in (mlp.gate, mlp.up))
            rows.append(torch.stack([g, u], dim=1).reshape(-1, width))   # 16 gate rows, 16 up rows, ...
        mo = m.heads * m.vdim
        c.nt_mix, c.nt_aux, c.nt_in = nt_mix, nt_aux, nt_mix + nt_aux + 2 * ff_tiles
        c.mix_k, c.act_k = _up(mo, kt), _up(16 * ff_tiles, kt)
        out = torch.zeros(width, c.mix_k + c.act_k, dtype=dtype, device=plain.device)
        out[:, :mo] = m.o
        if mlp is not None:
            out[:, c.mix_k:c.mix_k + mlp.down.shape[1]] = mlp.down
        w_in, w_out = pack_fragments(torch.cat(rows), dtype, width_pad), pack_fragments(out, dtype)
        self.keep += [w_in, w_out]
        c.w_in, c.w_out = w_in.data_ptr(), w_out.data_ptr()
        c.b_in = f32(None if bias is None else F.pad(bias, (0, 16 * nt_mix - bias.shape[0])))
        c.norm_w, c.heads, c.vdim = f32(layer.norm), m.heads, m.vdim
        if att:
            c.kind, c.kv_heads, c.dim, c.unit_rms, c.scale = 0, m.kv_heads, m.dim, int(m.unit_rms), m.scale
            big = max(m.dim, m.vdim)
            tiled = dtype == torch.bfloat16 and big <= 128               # the MFMA forms; other sizes and fp32 take the row kernel
            c.kp, c.vp = ((64 if big <= 64 else 128,) * 2) if tiled else (_up(m.dim, 8), _up(m.vdim, 8))
            c.r1, c.r2, c.pb, c.b_out = f32(m.r1), f32(m.r2), f32(m.pb), f32(m.o_bias)
        else:
            c.kind, c.groups, c.state, c.norm_groups, c.sp = 1, m.groups, m.state, m.norm_groups, _up(m.vdim, 4)
            c.taps = m.conv_w.shape[1]
            c.conv_w, c.conv_b, c.dt_bias, c.A_log, c.D, c.gnorm_w = (f32(t) for t in (m.conv_w.t(), m.conv_b, m.dt_bias, m.A_log, m.D, m.norm))

    def state_shapes(self, n_slots: int, max_len: int, dtype: torch.dtype) -> List[Tuple[tuple, torch.dtype]]:
        c = self.c
        if c.kind == 0:
            return [((n_slots, c.kv_heads, max_len, c.kp), dtype), ((n_slots, c.kv_heads, max_len, c.vp), dtype)]
        return [((n_slots, c.heads, c.state, c.sp), torch.float32),
                ((n_slots, c.taps, c.heads * c.vdim + 2 * c.groups * c.state), dtype)]


class StateSlots:
    """What requests keep between steps, ``n_slots`` of everything: one entry per layer run.  A request's first row (position 0) starts
    from nothing whatever its slot held before, so slots are handed out and taken back without clearing."""

    def __init__(self, decoder: "HybridDecoder", n_slots: int, max_len: int):
        self.decoder, self.n_slots, self.max_len = decoder, n_slots, max_len
        self.runs = [[torch.zeros(s, dtype=dt, device=decoder.device) for s, dt in decoder.packed[i].state_shapes(n_slots, max_len, decoder.dtype)]
                     for i, _ in decoder.runs]

    def grow(self, n_slots: int):
        """More slots; the live ones keep their contents and numbers."""
        for pair in self.runs:
            for k, t in enumerate(pair):
                n = torch.zeros((n_slots,) + tuple(t.shape[1:]), dtype=t.dtype, device=t.device)
                n[:self.n_slots] = t
                pair[k] = n
        self.n_slots = n_slots

    def bytes(self) -> int:
        return sum(t.numel() * t.element_size() for pair in self.runs for t in pair)


# ------------------------------------------------------------------------------------------------------------------- model --
class HybridDecoder:
    """The packed model: embedding (+ learned positions) -> layer runs -> norm -> head.  ``runs``: [(layer, add the embedding output
    first)] in execution order.  ``dtype`` torch.bfloat16 (serving) or torch.float32."""

    def __init__(self, *, layers: Sequence[HybridLayer], runs: Sequence[Tuple[int, bool]], embed: torch.Tensor, pos_embed: Optional[torch.Tensor],
                 final_norm: torch.Tensor, head: torch.Tensor, eps: float, norm_offset: float = 0.0, residual_mult: float = 1.0,
                 softcap: float = 0.0, max_positions: Optional[int] = None, dtype: torch.dtype = torch.bfloat16):
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError(f"hybrid decoders run in bfloat16 or float32, not {dtype}")
        if not embed.is_cuda:
            raise RuntimeError("HybridDecoder needs its weights on a ROCm GPU (no CPU fallback)")
        self.device, self.dtype = embed.device, dtype
        self.vocab_size, self.width = embed.shape
        self.width_pad = _up(self.width, k_tile(dtype))
        self.max_positions = max_positions if max_positions is not None else (pos_embed.shape[0] if pos_embed is not None else 1 << 20)
        self.eps, self.norm_offset, self.residual_mult, self.softcap = float(eps), float(norm_offset), float(residual_mult), float(softcap or 0.0)
        self.runs = [(int(i), bool(a)) for i, a in runs]
        self.packed = [_Packed(l, self.width, self.width_pad, dtype) for l in layers]
        self.embed = embed.to(dtype).contiguous()
        self.pos_embed = None if pos_embed is None else pos_embed.to(dtype).contiguous()
        self.final_norm = final_norm.float().contiguous()
        self.head = pack_fragments(head, dtype, self.width_pad)
        self._engines: Dict[tuple, object] = {}

    # what the framework's callers ask a model for
    def parameters(self):
        yield from (self.embed, self.final_norm, self.head)
        for p in self.packed:
            yield from p.keep

    def step_engine(self, n_slots: int, max_len: int, **kw) -> "HybridStep":
        return HybridStep(self, n_slots, max_len, **kw)

    @torch.no_grad()
    def forward(self, input_ids: torch.Tensor) -> torch.Tensor:
        """fp32 logits [B, S, vocab] of whole prompts."""
        B, S = input_ids.shape
        key = ("forward", B, S)
        if key not in self._engines:
            self._engines = {k: v for k, v in self._engines.items() if k[0] != "forward"}
            self._engines[key] = self.step_engine(B, S, max_rows=B * S)
        eng = self._engines[key]
        eng.launch([(b, 0, row, list(range(S))) for b, row in enumerate(input_ids.tolist())])
        return eng.logits[:B * S].view(B, S, self.vocab_size).clone()

    __call__ = forward

    @torch.no_grad()
    def generate(self, input_ids: torch.Tensor, max_new_tokens: int, eos_token_id=None, pad_token_id=None) -> torch.Tensor:
        """Greedy search as ``OneBitLlamaForCausalLM.generate`` (same arguments and result), one batcher slot per row."""
        from .serving import generate_batched
        return generate_batched(self, input_ids, max_new_tokens, eos_token_id, pad_token_id, self._engines)

    generate_native = generate


# ------------------------------------------------------------------------------------------------------------------- engine --
class HybridStep:
    """One scheduler step per ``launch``: ``(slot, start, tokens[, out])`` items as in ``MixedStep`` -- ``out`` = how many of the item's
    last rows are sampled (default 1) or the list of its rows that are -- to greedy tokens (device, one per sampled row in item order)
    and ``logits`` (fp32, same rows).  A step of single tokens replays a HIP graph captured per (row bucket, attention split plan)."""

    MAX_SPLITS = 64

    def __init__(self, model: HybridDecoder, n_slots: int, max_len: int, max_rows: int = 256, use_graph: bool = True):
        if n_slots < 1 or max_len < 1:
            raise ValueError("n_slots and max_len must be positive")
        if max_len > model.max_positions:
            raise ValueError(f"max_len {max_len} exceeds the model's {model.max_positions} positions")
        self.model, self.dev, self.max_len, self.use_graph = model, model.device, int(max_len), bool(use_graph)
        self.lib = _lib.load_hybrid()
        self.states = StateSlots(model, int(n_slots), self.max_len)
        self.logits = self.next_tokens = None
        self.launches = self.graph_launches = 0
        self._rows = self._outs = 0
        self._kv_heads = min([p.c.kv_heads for p in model.packed if p.c.kind == 0], default=1)
        self._bind()
        self._reserve(max(int(max_rows), 1), self.n_slots)

    @property
    def n_slots(self) -> int:
        return self.states.n_slots

    def grow(self, n_slots: int):
        """At least ``n_slots`` slots, live requests undisturbed."""
        if n_slots > self.n_slots:
            torch.cuda.synchronize(self.dev)
            self.states.grow(int(n_slots))
            self._bind()
            rows, outs = self._rows, self._outs
            self._rows = self._outs = 0
            self._reserve(rows, max(outs, self.n_slots))

    def _bind(self):
        m = self.model
        self._layers = (_HLayer * len(m.packed))(*[p.c for p in m.packed])
        self._runs = (_HRun * max(len(m.runs), 1))(*[_HRun(i, int(a), s[0].data_ptr(), s[1].data_ptr()) for (i, a), s in zip(m.runs, self.states.runs)])
        self._model = _HModel(ctypes.sizeof(_HModel), _lib.HYB_BF16 if m.dtype == torch.bfloat16 else _lib.HYB_F32, m.width, m.width_pad, m.vocab_size,
                              len(m.packed), len(m.runs), self.n_slots, self.max_len, m.max_positions, m.eps, m.norm_offset, m.residual_mult, m.softcap,
                              m.embed.data_ptr(), None if m.pos_embed is None else m.pos_embed.data_ptr(), m.final_norm.data_ptr(), m.head.data_ptr(),
                              self._layers, self._runs)
        self._stage = ItemStage(self.dev, self.n_slots, self.max_len, m.vocab_size)
        B = self.n_slots
        # single-token steps: [tokens | slot | position | offset | output rows] at a fixed device address (the graphs read it)
        self._g_stage = torch.zeros(5 * B, dtype=torch.int32, device=self.dev)
        self._g_host = [torch.zeros(5 * B, dtype=torch.int32).pin_memory() for _ in range(2)]
        self._g_np = [h.numpy() for h in self._g_host]
        self._g_ev, self._g_turn = [None, None], 0
        self._graphs: Dict[tuple, torch.cuda.CUDAGraph] = {}

    def _reserve(self, rows: int, outs: int):
        """Room for a step of ``rows`` token rows and ``outs`` sampled rows; grows geometrically, never shrinks (drops the graphs)."""
        if rows <= self._rows and outs <= self._outs:
            return
        rows = max(rows if rows <= self._rows else max(rows, 2 * self._rows), self._rows, self.n_slots, 64)
        outs = max(outs if outs <= self._outs else max(outs, 2 * self._outs), self._outs, self.n_slots)
        self._graphs = {}
        nb = int(self.lib.onebit_hybrid_workspace_bytes(ctypes.byref(self._model), rows, outs, self.n_slots, self.MAX_SPLITS))
        if nb == 0:
            raise ValueError("hybrid step: " + self.lib.onebit_hybrid_last_error().decode())
        self._ws = self.logits = None                              # (free the old blocks first)
        self._ws = torch.zeros(nb + 256, dtype=torch.uint8, device=self.dev)
        self._ws_off = (-self._ws.data_ptr()) % 256
        self.logits = torch.zeros(outs, self.model.vocab_size, dtype=torch.float32, device=self.dev)
        self.next_tokens = torch.zeros(outs, dtype=torch.int32, device=self.dev)
        self._stage.ensure(rows)
        self._rows, self._outs = rows, outs

    def _split_plan(self, rows: int, ctx: int) -> Tuple[int, int]:
        """(positions per workgroup, workgroups per head) of the decode attention: about four workgroups per CU, contexts in powers of
        two (one graph each), every context up to the bucket's end covered."""
        c = 256
        while c < ctx:
            c *= 2
        c = min(c, _up(self.max_len, 128))
        n = max(1, min(1024 // max(rows * self._kv_heads, 1), c // 128, self.MAX_SPLITS))
        chunk = _up(-(-c // n), 128)
        return chunk, -(-c // chunk)

    def _run(self, n_rows, n_dec, segs, n_out, plan, tokens, row_slot, row_pos, row_off, out_rows, residuals=None):
        seg_arr = (_HSeg * max(len(segs), 1))(*[_HSeg(*g) for g in segs])
        st = _HState(ctypes.sizeof(_HState), n_rows, n_dec, len(segs), n_out, plan[0], plan[1], tokens, row_slot, row_pos, row_off, seg_arr, out_rows,
                     self.logits.data_ptr(), self.next_tokens.data_ptr(), None if residuals is None else residuals.data_ptr(),
                     self._ws.data_ptr() + self._ws_off, self._ws.numel() - self._ws_off)
        with torch.cuda.device(self.dev):
            rc = self.lib.onebit_hybrid_step(ctypes.byref(self._model), ctypes.byref(st), self._rows, self._outs, self.n_slots, self.MAX_SPLITS,
                                             torch.cuda.current_stream(self.dev).cuda_stream)
        _lib.check_hybrid(rc, "onebit_hybrid_step")

    @torch.no_grad()
    def launch(self, items, residuals: bool = False):
        """Enqueue one step on the current stream; see the class.  ``residuals``: also return the residual stream after every layer run,
        fp32 [runs, rows, width] (rows in step order: single-token items first)."""
        n_out = sum((len(it[3]) if isinstance(it[3], (list, tuple)) else int(it[3])) if len(it) > 3 else 1 for it in items)
        if self.use_graph and not residuals and n_out == len(items) and all(len(it[2]) == 1 for it in items):
            return self._launch_graph(items)
        T = sum(len(it[2]) for it in items)
        self._reserve(T, max(n_out, T if residuals else 0))
        g = self._stage.stage(items)
        res = torch.empty(len(self.model.runs), T, self.model.width, dtype=torch.float32, device=self.dev) if residuals else None
        self._run(g.n_rows, g.n_dec, g.segs, g.n_out, self._split_plan(g.n_dec, g.dec_ctx) if g.n_dec else (128, 1), g.tokens, g.row_slot, g.row_pos,
                  g.row_off, g.out_rows, res)
        self.launches += 1
        return (self.next_tokens[:g.n_out], res) if residuals else self.next_tokens[:g.n_out]

    def _launch_graph(self, items):
        B, V = self.n_slots, self.model.vocab_size
        n = len(items)
        if not 0 < n <= B or len({it[0] for it in items}) != n:
            raise ValueError(f"step: {n} items for {B} slots, or a repeated slot")
        ctx = 0
        for i, (slot, start, toks) in enumerate(it[:3] for it in items):
            if not 0 <= slot < B or not 0 <= start < self.max_len or not 0 <= toks[0] < V:
                raise ValueError(f"step: item {i} (slot {slot}, start {start}, token {toks[0]}) outside the cache or the vocabulary")
            ctx = max(ctx, start + 1)
        rows = min(_up(n, 16), B)
        plan = self._split_plan(rows, ctx)
        graph = self._graphs.get((rows, plan))
        if graph is None:
            # warm-up on idle rows (loads the kernels; no slot's state moves), then record: the state advances once, by the replay
            self._stage_single([])
            base = self._g_stage.data_ptr()
            args = (rows, rows, [], rows, plan) + tuple(base + 4 * k * B for k in range(5))
            self._run(*args)
            torch.cuda.synchronize(self.dev)
            graph = torch.cuda.CUDAGraph()
            with torch.cuda.graph(graph):
                self._run(*args)
            self._graphs[(rows, plan)] = graph
        self._stage_single(items)
        graph.replay()
        self.launches += 1
        self.graph_launches += 1
        return self.next_tokens[:n]

    def _stage_single(self, items):
        """Single-token items into the row arrays the graphs read; the remaining rows are idle (no slot, no position)."""
        B, turn = self.n_slots, self._g_turn
        self._g_turn ^= 1
        if self._g_ev[turn] is not None:
            self._g_ev[turn].synchronize()
        st = self._g_np[turn]
        st[:] = 0
        st[B:3 * B] = -1
        st[4 * B:] = range(B)
        for i, it in enumerate(items):
            st[i], st[B + i], st[2 * B + i] = it[2][0], it[0], it[1]
        self._g_stage.copy_(self._g_host[turn], non_blocking=True)             # stream-ordered before the replay
        self._g_ev[turn] = torch.cuda.Event()
        self._g_ev[turn].record(torch.cuda.current_stream(self.dev))

    def step(self, items) -> List[int]:
        """``launch`` and wait: the greedy token of every sampled row."""
        return self.launch(items).tolist()
