"""Lebepel: a decoder-only model of sigmoid-attention and state-space layers with parallel feed-forwards, learned positions and a looped
stretch of layers.  This file reads its config.json and tensors and describes it with the parts of ``hybrid.py``; nothing here computes.

Per layer: h = rms(x) (1 + w), x += residual_mult (mixer(h) + ff(h)).  ``loop`` repeats a stretch of layers: every repetition keeps state
of its own, and from the second one on it starts by adding the embedding rows to the residual stream.  Logits are soft-capped."""
from __future__ import annotations

import json
import os
from dataclasses import dataclass, field
from typing import Dict, List, Optional, Tuple

import torch

from .hybrid import GatedFeedForward, HybridDecoder, HybridLayer, SigmoidAttention, StateSpace

ARCHITECTURE = "Lebepel"


@dataclass
class LebepelConfig:
    vocab_size: int
    width: int
    layers: List[dict]                         # {"type": "attention" | "mamba2", "mixer": {sizes}, "mlp": {"kind": "dense", "ff"} | None}
    norm_eps: float
    residual_mult: float
    logit_softcap: float
    max_positions: int
    loop: Optional[dict] = None                # {"start", "stop", "times"}
    extra: dict = field(default_factory=dict)

    _MIXER_KEYS = {"attention": ("heads", "kv_heads", "dim", "vdim", "scale"),
                   "mamba2": ("heads", "groups", "state", "vdim", "conv", "norm_groups")}

    def __post_init__(self):
        for i, lay in enumerate(self.layers):
            if lay.get("type") not in self._MIXER_KEYS:
                raise ValueError(f"layer {i}: mixer type {lay.get('type')!r}")
            missing = [k for k in self._MIXER_KEYS[lay["type"]] if k not in lay["mixer"]]
            if missing:
                raise ValueError(f"layer {i}: mixer without {missing}")
            if lay.get("mlp") is not None and lay["mlp"].get("kind") != "dense":
                raise ValueError(f"layer {i}: feed-forward kind {lay['mlp'].get('kind')!r}")
            m = lay["mixer"]
            if m["heads"] % (m["kv_heads"] if lay["type"] == "attention" else m["groups"]):
                raise ValueError(f"layer {i}: heads are not a multiple of their groups")
        if self.loop is not None and not (0 <= self.loop["start"] <= self.loop["stop"] <= len(self.layers) and self.loop["times"] >= 1):
            raise ValueError(f"loop {self.loop} does not fit {len(self.layers)} layers")

    @classmethod
    def from_dict(cls, raw: dict) -> "LebepelConfig":
        if raw.get("architecture") != ARCHITECTURE:
            raise ValueError(f"not a {ARCHITECTURE} config: architecture={raw.get('architecture')!r}")
        return cls(vocab_size=raw["vocab"], width=raw["width"], layers=raw["layers"], norm_eps=raw["norm"]["eps"],
                   residual_mult=raw.get("residual_mult", 1.0), logit_softcap=raw.get("logit_softcap") or 0.0, max_positions=raw["max_positions"],
                   loop=raw.get("loop"))

    def to_dict(self) -> dict:
        d = {"architecture": ARCHITECTURE, "layers": self.layers, "logit_softcap": self.logit_softcap, "max_positions": self.max_positions,
             "norm": {"eps": self.norm_eps}, "residual_mult": self.residual_mult, "vocab": self.vocab_size, "width": self.width}
        if self.loop is not None:
            d["loop"] = self.loop
        return d

    def runs(self) -> List[Tuple[int, bool]]:
        """Layer runs in execution order: (layer, add the embedding output to x first)."""
        n = len(self.layers)
        lp = self.loop or {"start": 0, "stop": 0, "times": 1}
        out = [(i, False) for i in range(lp["start"])]
        for p in range(lp["times"]):
            out += [(i, p > 0 and i == lp["start"]) for i in range(lp["start"], lp["stop"])]
        return out + [(i, False) for i in range(lp["stop"], n)]

    def tensor_shapes(self) -> Dict[str, tuple]:
        """Every tensor of a checkpoint of this configuration."""
        W = self.width
        s: Dict[str, tuple] = {"embed": (self.vocab_size, W), "pos": (self.max_positions, W), "final.norm": (W,), "head": (self.vocab_size, W)}
        for i, lay in enumerate(self.layers):
            m, p = lay["mixer"], f"l{i}."
            s[p + "norm1"] = (W,)
            if lay["type"] == "attention":
                for n, rows in (("q", m["heads"] * m["dim"]), ("k", m["kv_heads"] * m["dim"]), ("v", m["kv_heads"] * m["vdim"])):
                    s[p + f"mix.{n}"], s[p + f"mix.{n}.b"] = (rows, W), (rows,)
                s[p + "mix.o"], s[p + "mix.o.b"] = (W, m["heads"] * m["vdim"]), (W,)
                s.update({p + f"mix.{n}": (m["heads"],) for n in ("r1", "r2", "pb")})
            else:
                inner, ch = m["heads"] * m["vdim"], m["heads"] * m["vdim"] + 2 * m["groups"] * m["state"]
                s.update({p + "mix.in": (inner + ch + m["heads"], W), p + "mix.conv": (ch, m["conv"]), p + "mix.conv.b": (ch,),
                          p + "mix.norm": (inner,), p + "mix.o": (W, inner)})
                s.update({p + f"mix.{n}": (m["heads"],) for n in ("dt_bias", "A_log", "D")})
            if lay.get("mlp") is not None:
                ff = lay["mlp"]["ff"]
                s.update({p + "mlp.gate": (ff, W), p + "mlp.up": (ff, W), p + "mlp.down": (W, ff)})
        return s


class LebepelForCausalLM(HybridDecoder):
    def __init__(self, config: LebepelConfig, weights: Dict[str, torch.Tensor], dtype: torch.dtype = torch.bfloat16, device="cuda"):
        self.config = config
        for name, shape in config.tensor_shapes().items():
            if name not in weights:
                raise ValueError(f"checkpoint without tensor {name}")
            if tuple(weights[name].shape) != shape:
                raise ValueError(f"tensor {name}: shape {tuple(weights[name].shape)}, the configuration says {shape}")
        w = lambda n: weights[n].to(device)
        layers = []
        for i, lay in enumerate(config.layers):
            m, p = lay["mixer"], f"l{i}.mix."
            if lay["type"] == "attention":
                mixer = SigmoidAttention(m["heads"], m["kv_heads"], m["dim"], m["vdim"], float(m["scale"]), w(p + "q"), w(p + "k"), w(p + "v"), w(p + "o"),
                                         w(p + "q.b"), w(p + "k.b"), w(p + "v.b"), w(p + "o.b"), True, w(p + "r1"), w(p + "r2"), w(p + "pb"))
            else:
                mixer = StateSpace(m["heads"], m["groups"], m["state"], m["vdim"], m["norm_groups"], w(p + "in"), w(p + "conv"), w(p + "conv.b"),
                                   w(p + "dt_bias"), w(p + "A_log"), w(p + "D"), w(p + "norm"), w(p + "o"))
            q = f"l{i}.mlp."
            layers.append(HybridLayer(w(f"l{i}.norm1"), mixer, GatedFeedForward(w(q + "gate"), w(q + "up"), w(q + "down")) if lay.get("mlp") is not None else None))
        super().__init__(layers=layers, runs=config.runs(), embed=w("embed"), pos_embed=w("pos"), final_norm=w("final.norm"), head=w("head"),
                         eps=config.norm_eps, norm_offset=1.0, residual_mult=config.residual_mult, softcap=config.logit_softcap,
                         max_positions=config.max_positions, dtype=dtype)


def load(path: str, device="cuda", dtype: torch.dtype = torch.bfloat16) -> LebepelForCausalLM:
    """A model folder: config.json and model.safetensors."""
    from .checkpoint import read_safetensors
    with open(os.path.join(path, "config.json")) as f:
        cfg = LebepelConfig.from_dict(json.load(f))
    return LebepelForCausalLM(cfg, read_safetensors(os.path.join(path, "model.safetensors")), dtype, device)


def synthetic_weights(cfg: LebepelConfig, seed: int = 0, dtype=torch.bfloat16, device="cpu") -> Dict[str, torch.Tensor]:
    """Random weights of the configuration's shapes: linears N(0, 1 / fan_in), decays and step sizes in their usual ranges."""
    g = torch.Generator(device=device).manual_seed(seed)
    rnd = lambda *s: torch.randn(*s, generator=g, device=device)
    uni = lambda lo, hi, *s: lo + (hi - lo) * torch.rand(*s, generator=g, device=device)
    out = {}
    for name, shape in cfg.tensor_shapes().items():
        leaf = name.split(".", 1)[1] if name[0] == "l" and name[1].isdigit() else name
        if name in ("embed", "pos"):
            t = rnd(*shape) * (1.0 if name == "embed" else 0.3)
        elif leaf in ("norm1", "final.norm"):
            t = 0.1 * rnd(*shape)
        elif leaf == "mix.norm":
            t = 1 + 0.1 * rnd(*shape)
        elif leaf == "mix.r1":
            t = uni(0.3, 1.0, *shape)
        elif leaf == "mix.r2":
            t = uni(0.05, 0.5, *shape)
        elif leaf == "mix.pb":
            t = uni(-4.0, -2.0, *shape)
        elif leaf == "mix.A_log":
            t = uni(0.0, 1.5, *shape)
        elif leaf == "mix.dt_bias":
            t = uni(-4.0, -1.0, *shape)
        elif leaf == "mix.D":
            t = 1 + 0.2 * rnd(*shape)
        elif leaf == "mix.conv":
            t = rnd(*shape) / shape[1] ** 0.5
        elif len(shape) == 2:
            t = rnd(*shape) / shape[1] ** 0.5
        else:
            t = 0.1 * rnd(*shape)
        out[name] = t.to(dtype)
    return out


def build_synthetic_model(cfg: LebepelConfig, seed: int = 0, dtype=torch.bfloat16, device="cuda") -> LebepelForCausalLM:
    return LebepelForCausalLM(cfg, synthetic_weights(cfg, seed, torch.bfloat16, device), dtype, device)
