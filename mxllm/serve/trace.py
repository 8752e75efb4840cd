"""Trace replay: feed given token ids through a model step by step and write logits.

    bin/trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N   < steps.jsonl

Steps come on standard input, one JSON object a line:

    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": []}

``entries`` are each request's next tokens and the places among them whose logits are wanted;
requests in ``end`` give back their slot and cache after the step.  The logits of step n, in the
order of the entries and of ``want``, go to ``DIR/n.f32`` (little-endian f32, [wanted, vocab]), and
``done n`` to standard output.  Nothing is sampled; the model runs through ``Engine.prefill_batch``
and ``Engine.decode``, the engine's own prompt pass and (graphed) decode step.

A request's first entry is its prompt, all prompts of a step in one pass; later entries are decoded,
all requests of a step in one batch (entries of several tokens token by token).  ``float32``: weights,
activations and caches in f32, exit code 3 if the model's kernels are bf16 only.
"""
from __future__ import annotations

import argparse
import json
import os
import sys

import numpy as np
import torch

from ..models import build_model
from .engine import Engine

MAX_SLOTS = 256


class Replay:
    """Live requests of a trace on one engine."""

    def __init__(self, engine: Engine):
        self.eng = engine
        self.slot: dict[str, int] = {}

    def step(self, entries: list[dict], end: list[str]) -> torch.Tensor | None:
        """Run one step's entries; returns the wanted logits [n, vocab] f32 (None: none wanted)."""
        eng = self.eng
        rows: dict[tuple[int, int], torch.Tensor] = {}  # (entry, place) -> logits
        fresh = [(i, e) for i, e in enumerate(entries) if e["id"] not in self.slot]
        going = [(i, e) for i, e in enumerate(entries) if e["id"] in self.slot]
        if fresh:
            for _, e in fresh:
                s = self.slot[e["id"]] = eng.acquire()
                eng.extend(s, len(e["tokens"]) + 1)
            want = [list(e.get("want", ())) for _, e in fresh]
            logits = eng.prefill_batch([self.slot[e["id"]] for _, e in fresh], [e["tokens"] for _, e in fresh], want)
            rows.update(zip(((i, w) for (i, _), ws in zip(fresh, want) for w in ws), logits))
        for t in range(max((len(e["tokens"]) for _, e in going), default=0)):
            batch = [(i, e) for i, e in going if t < len(e["tokens"])]
            slots = [self.slot[e["id"]] for _, e in batch]
            for s in slots:
                eng.extend(s, eng.lens[s] + 1)
            logits = eng.decode(slots, torch.tensor([e["tokens"][t] for _, e in batch]))
            for b, (i, e) in enumerate(batch):
                if t in e.get("want", ()):
                    rows[i, t] = logits[b].float().clone()  # a graphed step's output is reused by the next
        for r in end:
            eng.release(self.slot.pop(r))
        out = [rows[i, w] for i, e in enumerate(entries) for w in e.get("want", ())]
        return torch.stack(out) if out else None


def replay(engine: Engine, lines, out_dir: str, say) -> None:
    rp = Replay(engine)
    for line in lines:
        if not line.strip():
            continue
        st = json.loads(line)
        logits = rp.step(st.get("entries", []), st.get("end", []))
        if logits is not None:
            a = logits.cpu().numpy().astype("<f4", copy=False)
            np.ascontiguousarray(a).tofile(os.path.join(out_dir, f"{st['step']}.f32"))
        say(f"done {st['step']}")


def make_engine(path: str, dtype: torch.dtype, max_tokens: int, device) -> Engine:
    torch.backends.cuda.matmul.allow_tf32 = False
    torch.set_float32_matmul_precision("highest")
    model = build_model(path, device=device, dtype=dtype).eval()
    slots = max(1, min(max_tokens, MAX_SLOTS))
    # live tokens, plus a partly filled block for every slot
    return Engine(model, max_batch=slots, max_seq=max_tokens + 8, kv_pool_tokens=max_tokens + 256 * slots)


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="trace_run", description=__doc__,
                                 formatter_class=argparse.RawDescriptionHelpFormatter)
    ap.add_argument("--model", required=True, help="directory with config.json and model.safetensors")
    ap.add_argument("--dtype", choices=["bfloat16", "float32"], default="bfloat16")
    ap.add_argument("--out", required=True, help="directory of the logits files")
    ap.add_argument("--max-tokens", type=int, required=True, help="most tokens that live requests hold at any time")
    a = ap.parse_args(argv)
    from ..models import MODEL_CLASSES, model_config

    dtype = getattr(torch, a.dtype)
    cls = MODEL_CLASSES[type(model_config(a.model))]
    if dtype == torch.float32 and not getattr(cls, "serves_float32", False):
        print("this model's kernels are bfloat16 only", file=sys.stderr)
        return 3
    from ..ops import _ext

    part = getattr(cls, "native_component", None)
    if part:
        _ext.load_component(part)  # compiles what the model needs if the checkout has no built library
    else:
        _ext.native()
    if not torch.cuda.is_available():
        print("trace_run needs a GPU", file=sys.stderr)
        return 1
    engine = make_engine(a.model, dtype, a.max_tokens, torch.device("cuda", 0))

    def say(text: str) -> None:
        sys.stdout.write(text + "\n")
        sys.stdout.flush()

    replay(engine, sys.stdin, a.out, say)
    return 0
