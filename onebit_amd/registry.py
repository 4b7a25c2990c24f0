"""Model families by config.json: which class loads a model folder, in which number formats it runs, and which native library it needs.

A family's ``engine`` is the step engine whose ``launch(items)`` runs one scheduler step (``MixedStep``, ``HybridStep``): what the batcher,
generation, evaluation and the trace runner drive."""
from __future__ import annotations

import json
import os
from dataclasses import dataclass
from typing import Callable, List, Optional

import torch

from . import build


@dataclass(frozen=True)
class Family:
    name: str
    matches: Callable[[dict], bool]                 # config.json -> is it this family?
    load: Callable                                  # (folder, device, dtype) -> model
    serving_dtype: torch.dtype                      # what its kernels serve in
    float32: bool                                   # do the step kernels also run in fp32?
    library: str                                    # native library built on demand
    engine: Callable                                # (model, slots, max_len) -> step engine with logits (launch, logits, n_slots)
    max_positions: Callable[[object], int]


def _load_onebit(path, device, dtype):
    from .checkpoint import load_inference_checkpoint
    return load_inference_checkpoint(path, device, dtype)


def _engine_onebit(model, n_slots, max_len):
    n_slots = max(n_slots, 32)                      # (a fixed cache: enough slots from the start)
    from .engine import MixedStep
    from .llama import KVCache
    cache = KVCache(model.config, n_slots, max_len, model.lm_head.weight.device, torch.float16)
    return MixedStep(model, cache.layers, n_slots, max_len, max_rows=64, keep_logits=True)


def _load_lebepel(path, device, dtype):
    from .lebepel import load
    return load(path, device, dtype)


def _load_serotar(path, device, dtype):
    from .serotar import load
    return load(path, device, dtype)


FAMILIES: List[Family] = [
    Family("serotar", lambda c: c.get("architecture") == "Serotar", _load_serotar, torch.bfloat16, True, build.LIB_HYBRID,
           lambda model, n, max_len: model.step_engine(n, max_len), lambda model: model.max_positions),
    Family("lebepel", lambda c: c.get("architecture") == "Lebepel", _load_lebepel, torch.bfloat16, True, build.LIB_HYBRID,
           lambda model, n, max_len: model.step_engine(n, max_len), lambda model: model.max_positions),
    Family("bitllama", lambda c: "architecture" not in c and c.get("model_type", "bitllama") == "bitllama", _load_onebit, torch.float16, False, build.LIB,
           _engine_onebit, lambda model: model.config.max_position_embeddings),
]


def register(family: Family):
    """Add a family (asked before the built-in ones)."""
    FAMILIES.insert(0, family)


def find_family(path: str) -> Family:
    with open(os.path.join(path, "config.json")) as f:
        raw = json.load(f)
    for fam in FAMILIES:
        if fam.matches(raw):
            return fam
    raise ValueError(f"{path}: no model family for architecture={raw.get('architecture')!r}, model_type={raw.get('model_type')!r}; "
                     f"known: {', '.join(f.name for f in FAMILIES)}")


def load_model(path: str, device="cuda", dtype: Optional[torch.dtype] = None):
    """The model of a folder, by its config.json; ``dtype`` None: the family's serving format."""
    fam = find_family(path)
    build.ensure(fam.library)
    return fam.load(path, device, fam.serving_dtype if dtype is None else dtype)
