"""Trace replay: a recorded schedule of steps run on the family's step engine and cache / state slots exactly as the batcher runs its own,
with logits instead of sampling.

One step per input line, as JSON:
  {"step": 7, "entries": [{"id": "req-1", "tokens": [11, 4], "want": [1]}, {"id": "req-2", "tokens": [9], "want": []}], "end": ["req-2"]}
An entry continues its request (or opens it) by ``tokens``; ``want`` indexes the tokens to report logits for; ``end`` frees the slots of the
requests it names once the step has run.  Reported logits go to OUT/<step>.f32 as raw little-endian fp32 rows of ``vocab`` values, entry by
entry; steps that report nothing write no file.  Each step is acknowledged with a line ``done <step>``."""
from __future__ import annotations

import json
import os
import sys
from typing import Dict, List, Optional, Tuple

import torch

from .registry import find_family, load_model
from .serving import SlotPool


class TraceSession:
    """Requests by name on the slots of a step engine: which slot each holds and how many tokens it has."""

    def __init__(self, family, model, max_len: int, n_slots: int = 8):
        self.engine = family.engine(model, n_slots, max_len)
        self.pool = SlotPool(self.engine.n_slots)
        self.live: Dict[str, Tuple[int, int]] = {}

    def step(self, entries: List[dict], end: List[str] = ()) -> Optional[torch.Tensor]:
        """One step of ``entries`` as one batch; fp32 logits [wanted, vocab] on the host, or None."""
        entries = [e for e in entries if e["tokens"]]
        new = sum(e["id"] not in self.live for e in entries)
        if new > len(self.pool):
            n = max(2 * self.pool.n, self.pool.n + new - len(self.pool))
            if not hasattr(self.engine, "grow"):
                raise RuntimeError(f"{self.pool.n} slots are taken and {type(self.engine).__name__} cannot grow")
            self.engine.grow(n)
            self.pool.grow(n)
        items = []
        for e in entries:
            slot, pos = self.live[e["id"]] if e["id"] in self.live else (self.pool.take(), 0)
            items.append((slot, pos, list(e["tokens"]), list(e["want"])))
            self.live[e["id"]] = (slot, pos + len(e["tokens"]))
        wanted = sum(len(it[3]) for it in items)
        out = None
        if items:
            # a step of single tokens samples every row anyway (one graph); the rows that are wanted are picked below
            single = all(len(it[2]) == 1 for it in items)
            self.engine.launch([it[:3] for it in items] if single else items)
            if wanted:
                rows = [i for i, it in enumerate(items) for _ in it[3]] if single else list(range(wanted))
                out = self.engine.logits[rows].float().cpu()
            elif torch.cuda.is_available():
                torch.cuda.synchronize()
        for rid in end:
            if rid in self.live:
                self.pool.give(self.live.pop(rid)[0])
        return out


def run(model_dir: str, dtype: str, out_dir: str, max_tokens: int, device: str = "cuda", lines=None, stdout=None) -> int:
    """The trace runner's main loop; returns the exit code (3: the family's kernels do not run in fp32)."""
    fam = find_family(model_dir)
    if dtype == "float32" and not fam.float32:
        print(f"{fam.name}: the step kernels do not run in float32", file=sys.stderr)
        return 3
    model = load_model(model_dir, device, torch.float32 if dtype == "float32" else None)
    session = TraceSession(fam, model, max(1, min(max_tokens, fam.max_positions(model))))
    os.makedirs(out_dir, exist_ok=True)
    stdout = stdout or sys.stdout
    for line in lines if lines is not None else sys.stdin:
        if not line.strip():
            continue
        st = json.loads(line)
        logits = session.step(st["entries"], st.get("end") or [])
        if logits is not None:
            part = os.path.join(out_dir, f".{st['step']}.part")
            with open(part, "wb") as f:
                f.write(logits.contiguous().numpy().astype("<f4").tobytes())
            os.replace(part, os.path.join(out_dir, f"{st['step']}.f32"))
        print(f"done {st['step']}", file=stdout, flush=True)
    return 0
