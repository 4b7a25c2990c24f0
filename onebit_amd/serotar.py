"""Serotar: a decoder-only model of latent-attention layers without positions, dense or mixture-of-experts feed-forwards, norms on the
sublayers' outputs only, a token input to every layer and an average over depth after it.  This file reads its config.json and tensors and
describes it with the parts of ``hybrid.py``; nothing here computes.

Embedding: scaled token row plus a row of a bigram table.  Per layer: x += ls1 n1(mixer(x)); x += ls2 n2(ff(x)); x += the token's own input;
x = sum_j dwa[j] X_j over the embedding output and all layer results.  The model's norm has ONE weight for all columns."""
from __future__ import annotations

import json
import os
from dataclasses import dataclass
from typing import Dict, List, Optional

import torch

from .hybrid import ExpertMixture, GatedFeedForward, HybridDecoder, HybridLayer, LatentAttention, TokenInput, XieluFeedForward

ARCHITECTURE = "Serotar"


@dataclass
class SerotarConfig:
    vocab_size: int
    width: int
    layers: List[dict]             # {"type": "latent_attention", "mixer": {sizes}, "mlp": {"kind": "dense" | "moe", ...} | None}
    norm_eps: float
    embed_scale: float = 1.0
    bigram: Optional[dict] = None  # {"buckets", "mul_prev", "mul_cur"}
    side_dim: int = 0              # columns of a layer's token input, 0: none

    _MIXER_KEYS = ("heads", "dim", "vdim", "q_rank", "kv_rank", "scale")

    def __post_init__(self):
        for i, lay in enumerate(self.layers):
            if lay.get("type") != "latent_attention":
                raise ValueError(f"layer {i}: mixer type {lay.get('type')!r}")
            missing = [k for k in self._MIXER_KEYS if k not in lay["mixer"]]
            if missing:
                raise ValueError(f"layer {i}: mixer without {missing}")
            mlp = lay.get("mlp")
            if mlp is None:
                continue
            if mlp.get("kind") not in ("dense", "moe"):
                raise ValueError(f"layer {i}: feed-forward kind {mlp.get('kind')!r}")
            if mlp["kind"] == "moe":
                r = mlp["router"]
                n, g = r["experts"] + r.get("identity", 0), r.get("groups") or {"count": 1, "keep": 1}
                if r["experts"] < 1 or g["count"] < 1 or n % g["count"] or not 1 <= g["keep"] <= g["count"] or not 1 <= r["top"] <= g["keep"] * (n // g["count"]):
                    raise ValueError(f"layer {i}: router {r}")

    @classmethod
    def from_dict(cls, raw: dict) -> "SerotarConfig":
        if raw.get("architecture") != ARCHITECTURE:
            raise ValueError(f"not a {ARCHITECTURE} config: architecture={raw.get('architecture')!r}")
        emb = raw.get("embedding") or {}
        return cls(vocab_size=raw["vocab"], width=raw["width"], layers=raw["layers"], norm_eps=raw["norm"]["eps"], embed_scale=emb.get("scale", 1.0),
                   bigram=emb.get("bigram"), side_dim=(raw.get("token_side") or {}).get("dim", 0))

    def to_dict(self) -> dict:
        emb = {"scale": self.embed_scale}
        if self.bigram:
            emb["bigram"] = self.bigram
        d = {"architecture": ARCHITECTURE, "embedding": emb, "layers": self.layers, "norm": {"eps": self.norm_eps}, "vocab": self.vocab_size, "width": self.width}
        if self.side_dim:
            d["token_side"] = {"dim": self.side_dim}
        return d

    def tensor_shapes(self) -> Dict[str, tuple]:
        """Every tensor of a checkpoint of this configuration."""
        W, n = self.width, len(self.layers)
        s: Dict[str, tuple] = {"embed": (self.vocab_size, W), "final.norm": (), "head": (self.vocab_size, W)}
        if self.bigram:
            s["bigram"] = (self.bigram["buckets"] + 1, W)
        if self.side_dim:
            s["side.embed"] = (self.vocab_size, n * self.side_dim)

        def gated(p, ff):
            s.update({p + "gate": (ff, W), p + "up": (ff, W), p + "down": (W, ff)})
        for i, lay in enumerate(self.layers):
            m, mlp, p = lay["mixer"], lay.get("mlp"), f"l{i}."
            s.update({p + "norm1": (), p + "ls1": (W,), p + "dwa": (i + 2,), p + "mix.dq": (m["q_rank"], W), p + "mix.dq.norm": (m["q_rank"],),
                      p + "mix.uq": (m["heads"] * m["dim"], m["q_rank"]), p + "mix.dkv": (m["kv_rank"], W), p + "mix.dkv.norm": (m["kv_rank"],),
                      p + "mix.uk": (m["heads"] * m["dim"], m["kv_rank"]), p + "mix.uv": (m["heads"] * m["vdim"], m["kv_rank"]),
                      p + "mix.o": (W, m["heads"] * m["vdim"])})
            if mlp is not None:
                s.update({p + "norm2": (), p + "ls2": (W,)})
                if mlp["kind"] == "dense":
                    s.update({p + "mlp.up": (mlp["ff"], W), p + "mlp.down": (W, mlp["ff"]), p + "mlp.act": (2,)})
                else:
                    r = mlp["router"]
                    total = r["experts"] + r.get("identity", 0)
                    s.update({p + "mlp.router": (total, W), p + "mlp.correction": (total,)})
                    for e in range(r["experts"]):
                        gated(p + f"mlp.e{e}.", mlp["expert"]["ff"])
                    if mlp.get("shared"):
                        gated(p + "mlp.shared.", mlp["shared"]["ff"])
            if self.side_dim:
                s.update({p + "side.gate": (self.side_dim, W), p + "side.proj": (W, self.side_dim), p + "side.norm": (W,)})
        return s


class SerotarForCausalLM(HybridDecoder):
    def __init__(self, config: SerotarConfig, weights: Dict[str, torch.Tensor], dtype: torch.dtype = torch.bfloat16, device="cuda"):
        self.config = config
        for name, shape in config.tensor_shapes().items():
            if name not in weights:
                raise ValueError(f"checkpoint without tensor {name}")
            if tuple(weights[name].shape) != shape and not (shape == () and weights[name].numel() == 1):
                raise ValueError(f"tensor {name}: shape {tuple(weights[name].shape)}, the configuration says {shape}")
        w = lambda n: weights[n].to(device)
        gated = lambda p: GatedFeedForward(w(p + "gate"), w(p + "up"), w(p + "down"))

        def out_norm(p, k):        # the norm's one weight and the layer scale behind it: one weight per column
            return w(p + f"norm{k}").float() * w(p + f"ls{k}").float()
        layers = []
        for i, lay in enumerate(config.layers):
            m, mlp, p = lay["mixer"], lay.get("mlp"), f"l{i}."
            q = p + "mix."
            mixer = LatentAttention(m["heads"], m["dim"], m["vdim"], float(m["scale"]), w(q + "dq"), w(q + "dq.norm"), w(q + "uq"), w(q + "dkv"),
                                    w(q + "dkv.norm"), w(q + "uk"), w(q + "uv"), w(q + "o"))
            ff, q = None, p + "mlp."
            if mlp is not None and mlp["kind"] == "dense":
                a = weights[q + "act"].float()
                ff = XieluFeedForward(w(q + "up"), w(q + "down"), float(a[0]), float(a[1]))
            elif mlp is not None:
                r = mlp["router"]
                g = r.get("groups") or {"count": 1, "keep": 1}
                ff = ExpertMixture([gated(q + f"e{e}.") for e in range(r["experts"])], w(q + "router"), w(q + "correction"), r["top"], r.get("identity", 0),
                                   g["count"], g["keep"], gated(q + "shared.") if mlp.get("shared") else None)
            side = TokenInput(w(p + "side.gate"), w(p + "side.proj"), w(p + "side.norm"), i * config.side_dim) if config.side_dim else None
            layers.append(HybridLayer(None, mixer, ff, sequential=True, mixer_out=out_norm(p, 1), mlp_out=None if ff is None else out_norm(p, 2),
                                      token_input=side, depth_average=w(p + "dwa")))
        b = config.bigram
        super().__init__(layers=layers, runs=[(i, False) for i in range(len(layers))], embed=w("embed"), pos_embed=None,
                         final_norm=w("final.norm").float().reshape(1).expand(config.width), head=w("head"), eps=config.norm_eps, dtype=dtype,
                         embed_scale=config.embed_scale, bigram=w("bigram") if b else None, bigram_mul=(b["mul_prev"], b["mul_cur"]) if b else (0, 0),
                         token_table=w("side.embed") if config.side_dim else None)


def load(path: str, device="cuda", dtype: torch.dtype = torch.bfloat16) -> SerotarForCausalLM:
    """A model folder: config.json and model.safetensors."""
    from .checkpoint import read_safetensors
    with open(os.path.join(path, "config.json")) as f:
        cfg = SerotarConfig.from_dict(json.load(f))
    return SerotarForCausalLM(cfg, read_safetensors(os.path.join(path, "model.safetensors")), dtype, device)


def synthetic_weights(cfg: SerotarConfig, seed: int = 0, dtype=torch.bfloat16, device="cpu") -> Dict[str, torch.Tensor]:
    """Random weights of the configuration's shapes: linears N(0, 1 / fan_in), norms and layer scales around one, depth weights around keeping the
    last result."""
    g = torch.Generator(device=device).manual_seed(seed)
    rnd = lambda *s: torch.randn(s, generator=g, device=device)
    out = {}
    for name, shape in cfg.tensor_shapes().items():
        leaf = name.rsplit(".", 1)[-1]
        if name in ("embed", "bigram", "side.embed"):
            t = rnd(*shape)
        elif leaf == "dwa":
            t = 0.2 * rnd(*shape)
            t[-1] += 1
        elif leaf in ("norm", "norm1", "norm2", "ls1", "ls2"):
            t = 1 + 0.1 * rnd(*shape)
        elif leaf == "correction":
            t = 0.1 * rnd(*shape) / shape[0] ** 0.5
        elif leaf == "act":
            t = 0.5 * rnd(*shape)
        else:
            t = rnd(*shape) / shape[-1] ** 0.5
        out[name] = t.to(dtype)
    return out


def build_synthetic_model(cfg: SerotarConfig, seed: int = 0, dtype=torch.bfloat16, device="cuda") -> SerotarForCausalLM:
    return SerotarForCausalLM(cfg, synthetic_weights(cfg, seed, torch.bfloat16, device), dtype, device)
