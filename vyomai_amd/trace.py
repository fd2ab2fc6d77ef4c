"""Trace replay: given token ids go through a model step by step, on the model's own prefill / decode path and cache, and
the logits at chosen places are written out.  Nothing is sampled.

Steps are read from standard input, one JSON object a line:

    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": []}

entries: the next tokens of each request and the places among them whose logits are wanted; all entries of a step are one
batch.  end: requests that give their cache slot back after this step.  A step with wanted places writes OUT/<step>.f32
(float32 little-endian, [wanted, vocab], in the order of the entries), and every step prints 'done <step>'.
"""
from __future__ import annotations

import argparse
import json
import os
import sys
from typing import Dict, List

import torch

DTYPES = {"bfloat16": torch.bfloat16, "float32": torch.float32}


class TraceSession:
    """Requests by name over one model and one SlotCache."""

    def __init__(self, model, capacity: int = 64) -> None:
        self.model, self.cache = model, model.new_cache(1, capacity)
        self.slot: Dict[str, int] = {}

    @torch.no_grad()
    def step(self, entries: List[dict], end: List[str]) -> torch.Tensor:
        """-> logits (wanted, vocab) of the step."""
        model, cache = self.model, self.cache
        for e in entries:
            if e["id"] not in self.slot:
                self.slot[e["id"]] = cache.allocate(1)[0]
        slots = [self.slot[e["id"]] for e in entries]
        counts = [len(e["tokens"]) for e in entries]
        out = torch.empty(0, model.vocab)
        if entries:
            L = max(counts)
            tokens = torch.tensor([e["tokens"] + [0] * (L - len(e["tokens"])) for e in entries], dtype=torch.long,
                                  device=model.device)
            want = [b * L + w for b, e in enumerate(entries) for w in e["want"]]
            if L == 1:
                logits = model.decode(tokens.view(-1), cache, slots)
            else:
                hidden = model.prefill(tokens, counts, cache, slots).view(len(entries) * L, -1)
                logits = None
            if want:
                rows = torch.tensor(want, device=model.device)
                logits = logits.index_select(0, rows) if logits is not None else model.logits(hidden.index_select(0, rows))
                out = logits.float().cpu()
        cache.free([self.slot.pop(i) for i in end])
        return out


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="trace_run", description="Replay a trace of token ids and write logits.")
    ap.add_argument("--model", required=True, help="folder with config.json and *.safetensors")
    ap.add_argument("--dtype", required=True, choices=sorted(DTYPES))
    ap.add_argument("--out", required=True, help="folder for <step>.f32")
    ap.add_argument("--max-tokens", type=int, default=0, help="most tokens that live requests hold at any time (a hint)")
    a = ap.parse_args(argv)
    from .models.registry import load_pretrained
    session = TraceSession(load_pretrained(a.model, DTYPES[a.dtype]))
    for line in sys.stdin:
        if not line.strip():
            continue
        s = json.loads(line)
        logits = session.step(s["entries"], s.get("end", []))
        if logits.shape[0]:
            part = os.path.join(a.out, f".{s['step']}.part")
            logits.contiguous().numpy().astype("<f4").tofile(part)
            os.replace(part, os.path.join(a.out, f"{s['step']}.f32"))
        print(f"done {s['step']}", flush=True)
    return 0
