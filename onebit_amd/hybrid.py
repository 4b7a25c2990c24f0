"""Hybrid decoders: dense-weight decoder-only models whose layers mix different sequence mixers, on ``libonebit_hybrid.so``
(include/onebit_hybrid.h).

A design describes itself with the parts below -- ``SigmoidAttention`` / ``StateSpace`` / ``LatentAttention`` mixers, ``GatedFeedForward`` /
``XieluFeedForward`` / ``ExpertMixture``, ``TokenInput``, ``HybridLayer``, the order of layer runs -- and inherits packing, cache / state, the
step engine, generation and evaluation from ``HybridDecoder``.
A PARALLEL layer is  x += mult * (mixer(norm(x)) + ff(norm(x)))  as two matrix products: mixer and feed-forward read one normalised row, so
their input projections are ONE weight matrix, and their output projections act on disjoint column ranges of one row, so they are one matrix
too (csrc/ob_dense.h has the packed layout).  A SEQUENTIAL layer runs them one after the other, each with optional norms on its input and on
its output, then optionally adds the token's own input and averages over depth.

``StateSlots`` holds what requests leave between steps, per layer RUN (a layer that a loop repeats has an entry for each repetition): keys and
values, latent rows, or the fp32 recurrent state and the ring of convolution inputs; and, where the embedding looks at the token before, the
slots' tokens.  ``HybridStep`` is the step engine with ``MixedStep``'s
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


class _HLatent(ctypes.Structure):
    _fields_ = [("q_rank", _i32), ("kv_rank", _i32), ("nt_q", _i32), ("rp", _i32), ("tiled", _i32), ("flash", _i32), ("vdp", _i32), ("qn_w", _vp),
                ("kvn_w", _vp), ("w_uq", _vp), ("w_uk", _vp), ("w_uv", _vp), ("w_kv", _vp)]


class _HFf(ctypes.Structure):
    _fields_ = [("nt_plain", _i32), ("nt_gated", _i32), ("nt_aux", _i32), ("nt_expert", _i32), ("experts", _i32), ("identity", _i32), ("top", _i32),
                ("groups", _i32), ("keep", _i32), ("act_a", _f), ("act_b", _f), ("w_plain_in", _vp), ("w_plain_out", _vp), ("w_gated_in", _vp),
                ("w_gated_out", _vp), ("w_expert_in", _vp), ("w_expert_out", _vp), ("correction", _vp)]


class _HSide(ctypes.Structure):
    _fields_ = [("dim", _i32), ("nt", _i32), ("w_gate", _vp), ("w_proj", _vp), ("norm_w", _vp), ("table", _vp)]


class _HLayer(ctypes.Structure):
    _fields_ = [("kind", _i32), ("nt_mix", _i32), ("nt_aux", _i32), ("nt_in", _i32), ("mix_k", _i32), ("act_k", _i32),
                ("w_in", _vp), ("w_out", _vp), ("b_in", _vp), ("b_out", _vp), ("norm_w", _vp), ("heads", _i32), ("vdim", _i32),
                ("kv_heads", _i32), ("dim", _i32), ("kp", _i32), ("vp", _i32), ("unit_rms", _i32), ("scale", _f),
                ("r1", _vp), ("r2", _vp), ("pb", _vp),
                ("groups", _i32), ("state", _i32), ("taps", _i32), ("norm_groups", _i32), ("sp", _i32),
                ("conv_w", _vp), ("conv_b", _vp), ("dt_bias", _vp), ("A_log", _vp), ("D", _vp), ("gnorm_w", _vp),
                ("form", _i32), ("post1_w", _vp), ("pre2_w", _vp), ("post2_w", _vp), ("dwa", _vp), ("latent", _HLatent), ("ff", _HFf), ("side", _HSide)]


class _HRun(ctypes.Structure):
    _fields_ = [("layer", _i32), ("add_embedding", _i32), ("s0", _vp), ("s1", _vp)]


class _HModel(ctypes.Structure):
    _fields_ = [("struct_size", _u64), ("dtype", _i32), ("width", _i32), ("width_pad", _i32), ("vocab", _i32), ("n_layers", _i32),
                ("n_runs", _i32), ("n_slots", _i32), ("max_len", _i32), ("max_pos", _i32), ("eps", _f), ("norm_off", _f), ("mult", _f),
                ("softcap", _f), ("embed", _vp), ("pos_embed", _vp), ("final_norm", _vp), ("head", _vp),
                ("layers", ctypes.POINTER(_HLayer)), ("runs", ctypes.POINTER(_HRun)), ("embed_scale", _f), ("bigram", _vp), ("buckets", _i32),
                ("mul_prev", _i32), ("mul_cur", _i32), ("token_history", _vp), ("side_cols", _i32)]


class _HSeg(ctypes.Structure):
    _fields_ = [("row0", _i32), ("n", _i32), ("slot", _i32), ("past", _i32)]


class _HState(ctypes.Structure):
    _fields_ = [("struct_size", _u64), ("n_rows", _i32), ("n_dec", _i32), ("n_seg", _i32), ("n_out", _i32), ("n_short", _i32), ("attn_chunk", _i32),
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
class LatentAttention:
    """Softmax attention whose keys and values are projections of one normalised vector c per token (only c is cached), without positions:
    q = uq rms(dq h) dq_norm, c = rms(dkv h) dkv_norm, per head k = uk c, v = uv c, score = q.k scale."""
    heads: int
    dim: int
    vdim: int
    scale: float
    dq: torch.Tensor
    dq_norm: torch.Tensor
    uq: torch.Tensor              # [heads dim, q_rank]
    dkv: torch.Tensor
    dkv_norm: torch.Tensor
    uk: torch.Tensor              # [heads dim, kv_rank]
    uv: torch.Tensor              # [heads vdim, kv_rank]
    o: torch.Tensor


@dataclass
class XieluFeedForward:
    """down(f(up h)), f(z) = softplus(p) z^2 + z / 2 above zero, (1/2 + softplus(q)) (e^z - 1 - z) + z / 2 below."""
    up: torch.Tensor
    down: torch.Tensor
    p: float
    q: float


@dataclass
class ExpertMixture:
    """Routed gated feed-forwards: softmax scores over experts and ``identity`` trailing experts that return their input; the ``top`` largest
    scores + correction among the ``keep`` best of ``groups`` equal groups of neighbours are used, weighted by their plain scores;
    ``shared`` runs for every token."""
    experts: List[GatedFeedForward]
    router: torch.Tensor          # [experts + identity, width]
    correction: torch.Tensor
    top: int
    identity: int = 0
    groups: int = 1
    keep: int = 1
    shared: Optional[GatedFeedForward] = None


@dataclass
class TokenInput:
    """x += rms(proj(gelu_tanh(gate x) * e)) norm, e = columns ``column`` .. of the token's row in the model's ``token_table``."""
    gate: torch.Tensor
    proj: torch.Tensor
    norm: torch.Tensor
    column: int


@dataclass
class HybridLayer:
    """``sequential`` False: the parallel form, ``norm`` in front of both.  True: mixer, then feed-forward; ``norm`` / ``mlp_norm`` on their inputs and
    ``mixer_out`` / ``mlp_out`` on their outputs are RMS norms with these weights per column, None: no norm there.  ``depth_average``: weights
    over the embedding output and the results of the layer runs up to this one."""
    norm: Optional[torch.Tensor]
    mixer: object
    mlp: Optional[object]
    sequential: bool = False
    mixer_out: Optional[torch.Tensor] = None
    mlp_norm: Optional[torch.Tensor] = None
    mlp_out: Optional[torch.Tensor] = None
    token_input: Optional[TokenInput] = None
    depth_average: Optional[torch.Tensor] = None


def _gate_up(ff: GatedFeedForward, tiles: int) -> torch.Tensor:
    """Rows [16 of gate, 16 of up, ...], ``tiles`` tiles of each."""
    g, u = (_pad_rows(t, 16 * tiles).view(tiles, 16, -1) for t in (ff.gate, ff.up))
    return torch.stack([g, u], dim=1).reshape(32 * tiles, -1)


class _Packed:
    """A layer on the device: its fragment-major matrices and everything else as fp32 vectors, behind a filled ``_HLayer``."""

    def __init__(self, layer: HybridLayer, width: int, width_pad: int, dtype: torch.dtype, token_table: Optional[torch.Tensor] = None):
        self.dtype, self.width, self.width_pad = dtype, width, width_pad
        m, mlp = layer.mixer, layer.mlp
        self.keep: List[torch.Tensor] = []
        c = self.c = _HLayer()
        c.heads, c.vdim, c.norm_w = m.heads, m.vdim, self._f32(layer.norm)
        merged = None
        if layer.sequential:
            c.form = 1
            c.post1_w, c.pre2_w, c.post2_w = self._f32(layer.mixer_out), self._f32(layer.mlp_norm), self._f32(layer.mlp_out)
            self._feed_forward(mlp)
        else:
            if layer.norm is None or any(t is not None for t in (layer.mixer_out, layer.mlp_norm, layer.mlp_out, layer.token_input)):
                raise ValueError("a parallel layer has one norm, in front of both parts")
            if mlp is not None and not isinstance(mlp, GatedFeedForward):
                raise ValueError(f"a parallel layer's feed-forward is gated, not {type(mlp).__name__}")
            merged = mlp
        if layer.token_input is not None:
            self._token_input(layer.token_input, token_table)
        c.dwa = self._f32(layer.depth_average)
        if isinstance(m, LatentAttention):
            if not layer.sequential:
                raise ValueError("latent attention needs a sequential layer")
            self._latent(m)
        else:
            self._merged(m, merged)

    def _f32(self, t):
        if t is None:
            return None
        t = t.detach().float().contiguous()
        self.keep.append(t)
        return t.data_ptr()

    def _pack(self, w, k_pad=None):
        p = pack_fragments(w, self.dtype, k_pad)
        self.keep.append(p)
        return p.data_ptr()

    def _merged(self, m, mlp):
        """Sigmoid attention or state space: [mixer projections | gate / up of a parallel layer] and [mixer output | down]."""
        c, dtype, kt, f32 = self.c, self.dtype, k_tile(self.dtype), self._f32
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
            rows.append(_gate_up(mlp, ff_tiles))
        mo = m.heads * m.vdim
        c.nt_mix, c.nt_aux, c.nt_in = nt_mix, nt_aux, nt_mix + nt_aux + 2 * ff_tiles
        c.mix_k, c.act_k = _up(mo, kt), _up(16 * ff_tiles, kt)
        out = torch.zeros(self.width, c.mix_k + c.act_k, dtype=dtype, device=plain.device)
        out[:, :mo] = m.o
        if mlp is not None:
            out[:, c.mix_k:c.mix_k + mlp.down.shape[1]] = mlp.down
        c.w_in, c.w_out = self._pack(torch.cat(rows), self.width_pad), self._pack(out)
        c.b_in = f32(None if bias is None else F.pad(bias, (0, 16 * nt_mix - bias.shape[0])))
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

    def _latent(self, m: LatentAttention):
        c, l, H, kt = self.c, self.c.latent, m.heads, k_tile(self.dtype)
        c.kind, c.dim, c.scale = 2, m.dim, m.scale
        l.q_rank, l.kv_rank = m.dq.shape[0], m.dkv.shape[0]
        bf, big = self.dtype == torch.bfloat16, max(m.dim, m.vdim)
        l.tiled = int(bf and l.kv_rank <= 512)
        l.flash = int(l.tiled and big <= 128)
        l.rp = next(n for n in (64, 128, 256, 512) if n >= l.kv_rank) if l.tiled else _up(l.kv_rank, 32)
        c.kp = c.vp = (64 if big <= 64 else 128) if l.flash else _up(m.dim, 32)
        l.vdp = _up(m.vdim, 32)
        l.nt_q = -(-l.q_rank // 16)
        rows = torch.cat([_pad_rows(m.dq, 16 * l.nt_q), _pad_rows(m.dkv, _up(l.kv_rank, 16))])
        c.nt_mix = c.nt_in = rows.shape[0] // 16
        c.w_in = self._pack(rows, self.width_pad)
        heads = lambda w, n, p: F.pad(w.view(H, n, -1), (0, 0, 0, p - n))                  # [heads, p, rank], rows beyond n zero
        l.w_uq = self._pack(heads(m.uq, m.dim, c.kp).reshape(H * c.kp, -1))
        uk, uv = heads(m.uk, m.dim, c.kp), heads(m.uv, m.vdim, l.vdp)
        l.w_uk = self._pack(F.pad(uk.transpose(1, 2), (0, 0, 0, l.rp - l.kv_rank)).reshape(H * l.rp, c.kp))
        l.w_uv = self._pack(uv.reshape(H * l.vdp, -1), l.rp)
        if l.flash:
            l.w_kv = self._pack(torch.cat([uk, heads(m.uv, m.vdim, c.kp)]).reshape(2 * H * c.kp, -1), l.rp)
        l.qn_w, l.kvn_w = self._f32(m.dq_norm), self._f32(m.dkv_norm)
        c.mix_k = _up(H * l.vdp, kt)
        c.w_out = self._pack(F.pad(m.o.view(self.width, H, m.vdim), (0, l.vdp - m.vdim)).reshape(self.width, -1), c.mix_k)

    def _feed_forward(self, mlp):
        f = self.c.ff
        if mlp is None:
            return
        if isinstance(mlp, XieluFeedForward):
            f.nt_plain = _up(mlp.up.shape[0], 32) // 16
            f.w_plain_in, f.w_plain_out = self._pack(_pad_rows(mlp.up, 16 * f.nt_plain), self.width_pad), self._pack(mlp.down, 16 * f.nt_plain)
            f.act_a = float(F.softplus(torch.tensor(mlp.p, dtype=torch.float64)))
            f.act_b = 0.5 + float(F.softplus(torch.tensor(mlp.q, dtype=torch.float64)))
            return
        mix = mlp if isinstance(mlp, ExpertMixture) else None
        gated = mlp if mix is None else mix.shared
        rows = []
        if mix is not None:
            E = len(mix.experts)
            f.experts, f.identity, f.top, f.groups, f.keep = E, mix.identity, mix.top, mix.groups, mix.keep
            if mix.router.shape[0] != E + mix.identity:
                raise ValueError(f"router of {mix.router.shape[0]} rows for {E} experts and {mix.identity} identity experts")
            f.nt_aux = _up(E + mix.identity, 32) // 16
            rows.append(_pad_rows(mix.router, 16 * f.nt_aux))
            f.correction = self._f32(mix.correction)
            tiles = _up(mix.experts[0].gate.shape[0], 32) // 16
            f.nt_expert = 2 * tiles
            f.w_expert_in = self._pack(torch.cat([_gate_up(e, tiles) for e in mix.experts]), self.width_pad)
            down = torch.zeros(E, _up(self.width, 16), 16 * tiles, dtype=self.dtype, device=mix.router.device)
            for i, e in enumerate(mix.experts):
                down[i, :self.width, :e.down.shape[1]] = e.down
            f.w_expert_out = self._pack(down.view(-1, 16 * tiles))
        if gated is not None:
            tiles = _up(gated.gate.shape[0], 32) // 16
            f.nt_gated = 2 * tiles
            rows.append(_gate_up(gated, tiles))
            f.w_gated_out = self._pack(gated.down, 16 * tiles)
        f.w_gated_in = self._pack(torch.cat(rows), self.width_pad)

    def _token_input(self, t: TokenInput, table: torch.Tensor):
        s = self.c.side
        s.dim = t.gate.shape[0]
        if table is None or not 0 <= t.column <= table.shape[1] - s.dim:
            raise ValueError(f"token input: columns {t.column} .. {t.column + s.dim} of the token table")
        s.nt = _up(s.dim, 32) // 16
        s.w_gate, s.w_proj, s.norm_w = self._pack(_pad_rows(t.gate, 16 * s.nt), self.width_pad), self._pack(t.proj, 16 * s.nt), self._f32(t.norm)
        s.table = table.data_ptr() + t.column * table.element_size()

    def state_shapes(self, n_slots: int, max_len: int, dtype: torch.dtype) -> List[Tuple[tuple, torch.dtype]]:
        c = self.c
        if c.kind == 0:
            return [((n_slots, c.kv_heads, max_len, c.kp), dtype), ((n_slots, c.kv_heads, max_len, c.vp), dtype)]
        if c.kind == 2:
            kt = k_tile(dtype)
            return [((n_slots, -(-max_len // 16), c.latent.rp // kt, 64, kt // 4), dtype)]
        return [((n_slots, c.heads, c.state, c.sp), torch.float32),
                ((n_slots, c.taps, c.heads * c.vdim + 2 * c.groups * c.state), dtype)]


class StateSlots:
    """What requests keep between steps, ``n_slots`` of everything: one entry per layer run.  A request's first row (position 0) starts
    from nothing whatever its slot held before, so slots are handed out and taken back without clearing."""

    def __init__(self, decoder: "HybridDecoder", n_slots: int, max_len: int):
        self.decoder, self.n_slots, self.max_len = decoder, n_slots, max_len
        self.runs = [[torch.zeros(s, dtype=dt, device=decoder.device) for s, dt in decoder.packed[i].state_shapes(n_slots, max_len, decoder.dtype)]
                     for i, _ in decoder.runs]
        self.tokens = torch.zeros(n_slots, max_len, dtype=torch.int32, device=decoder.device) if decoder.bigram is not None else None

    def grow(self, n_slots: int):
        """More slots; the live ones keep their contents and numbers."""
        def more(t):
            n = torch.zeros((n_slots,) + tuple(t.shape[1:]), dtype=t.dtype, device=t.device)
            n[:self.n_slots] = t
            return n
        for pair in self.runs:
            pair[:] = [more(t) for t in pair]
        if self.tokens is not None:
            self.tokens = more(self.tokens)
        self.n_slots = n_slots

    def bytes(self) -> int:
        return sum(t.numel() * t.element_size() for pair in self.runs for t in pair)


# ------------------------------------------------------------------------------------------------------------------- model --
class HybridDecoder:
    """The packed model: embedding (+ learned positions, + bigram rows) -> layer runs -> norm -> head.  ``runs``: [(layer, add the embedding
    output first)] in execution order.  ``bigram`` [buckets + 1, width] with ``bigram_mul`` (previous, current): row (previous token a + token b) %
    buckets is added to the scaled embedding, the last row at position 0.  ``dtype`` torch.bfloat16 (serving) or torch.float32."""

    def __init__(self, *, layers: Sequence[HybridLayer], runs: Sequence[Tuple[int, bool]], embed: torch.Tensor, pos_embed: Optional[torch.Tensor],
                 final_norm: torch.Tensor, head: torch.Tensor, eps: float, norm_offset: float = 0.0, residual_mult: float = 1.0,
                 softcap: float = 0.0, max_positions: Optional[int] = None, dtype: torch.dtype = torch.bfloat16, embed_scale: float = 1.0,
                 bigram: Optional[torch.Tensor] = None, bigram_mul: Tuple[int, int] = (0, 0), token_table: Optional[torch.Tensor] = None):
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
        self.token_table = None if token_table is None else token_table.to(dtype).contiguous()
        self.packed = [_Packed(l, self.width, self.width_pad, dtype, self.token_table) for l in layers]
        for r, (i, _) in enumerate(self.runs):
            d = layers[i].depth_average
            if d is not None and d.shape != (r + 2,):
                raise ValueError(f"layer run {r}: a depth average over {tuple(d.shape)} of {r + 2} results")
        self.embed_scale = float(embed_scale)
        self.bigram = None if bigram is None else bigram.to(dtype).contiguous()
        self.bigram_mul = (0, 0) if bigram is None else tuple(int(v) % (bigram.shape[0] - 1) for v in bigram_mul)      # (the row is taken modulo the buckets)
        self.embed = embed.to(dtype).contiguous()
        self.pos_embed = None if pos_embed is None else pos_embed.to(dtype).contiguous()
        self.final_norm = final_norm.float().contiguous()
        self.head = pack_fragments(head, dtype, self.width_pad)
        self._engines: Dict[tuple, object] = {}

    # what the framework's callers ask a model for
    def parameters(self):
        yield from (t for t in (self.embed, self.final_norm, self.head, self.pos_embed, self.bigram, self.token_table) if t is not None)
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
        self._runs = (_HRun * max(len(m.runs), 1))(*[_HRun(i, int(a), s[0].data_ptr(), s[1].data_ptr() if len(s) > 1 else None)
                                                     for (i, a), s in zip(m.runs, self.states.runs)])
        self._model = _HModel(ctypes.sizeof(_HModel), _lib.HYB_BF16 if m.dtype == torch.bfloat16 else _lib.HYB_F32, m.width, m.width_pad, m.vocab_size,
                              len(m.packed), len(m.runs), self.n_slots, self.max_len, m.max_positions, m.eps, m.norm_offset, m.residual_mult, m.softcap,
                              m.embed.data_ptr(), None if m.pos_embed is None else m.pos_embed.data_ptr(), m.final_norm.data_ptr(), m.head.data_ptr(),
                              self._layers, self._runs, m.embed_scale, None if m.bigram is None else m.bigram.data_ptr(),
                              0 if m.bigram is None else m.bigram.shape[0] - 1, *m.bigram_mul, None if m.bigram is None else self.states.tokens.data_ptr(),
                              0 if m.token_table is None else m.token_table.shape[1])
        self._stage = ItemStage(self.dev, self.n_slots, self.max_len, m.vocab_size, short=_lib.HYB_SHORT)
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

    def _run(self, n_rows, n_dec, segs, n_out, n_short, plan, tokens, row_slot, row_pos, row_off, out_rows, residuals=None):
        seg_arr = (_HSeg * max(len(segs), 1))(*[_HSeg(*g) for g in segs])
        st = _HState(ctypes.sizeof(_HState), n_rows, n_dec, len(segs), n_out, n_short, plan[0], plan[1], tokens, row_slot, row_pos, row_off, seg_arr, out_rows,
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
        self._run(g.n_rows, g.n_dec, g.segs, g.n_out, g.n_short, self._split_plan(max(g.n_dec, 1), g.dec_ctx) if g.n_dec or g.n_short else (128, 1), g.tokens, g.row_slot, g.row_pos,
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
            args = (rows, rows, [], rows, 0, plan) + tuple(base + 4 * k * B for k in range(5))
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
