"""Trace runner: feed given token ids through a model step by step and write logits.

    bin/trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N < steps.jsonl

One JSON object per input line: {"step": n, "entries": [{"id", "tokens", "want"}], "end": [ids]}.
The entries of a step are one batch: either new requests (their first tokens) or live requests that
all go on by the same number of tokens. Logits at the wanted places are written to OUT/<step>.f32
(little-endian fp32, [wanted, vocab], in the order of the entries and of `want`), and `done <step>`
is printed after every step. Runs the model step, cache and kernels of `models.generation`: new
requests are left-padded into one KVCache, later steps continue it, and the rows of ended requests
leave it.
"""
from __future__ import annotations

import argparse
import json
import os
import sys
from typing import Dict, List, Optional

import torch

from ..models.generation import KVCache
from ..models.loader import load_causal_lm


class _Batch:
    """Requests that started together: cache row r belongs to ids[r]."""

    def __init__(self, ids: List[str], cache: KVCache):
        self.ids, self.cache = ids, cache

    def split(self, ids: List[str]) -> "_Batch":
        return _Batch(ids, self.cache.keep_rows([self.ids.index(i) for i in ids]))


class TraceRunner:
    def __init__(self, model, max_tokens: Optional[int] = None):
        self.model = model
        self.max_tokens = max_tokens
        self.where: Dict[str, _Batch] = {}

    def _start(self, ids, toks, device):
        B, T = len(ids), max(len(t) for t in toks)
        inp = torch.zeros((B, T), dtype=torch.long)
        for r, t in enumerate(toks):
            inp[r, T - len(t):] = torch.tensor(t)
        start = torch.tensor([T - len(t) for t in toks], dtype=torch.int32, device=device)
        room = T + 64 if self.max_tokens is None else min(max(T, self.max_tokens), T + 1024)
        b = _Batch(ids, KVCache(self.model, B, room, start))
        for i in ids:
            self.where[i] = b
        return b, inp.to(device)

    def _go_on(self, ids, toks, device):
        b = self.where[ids[0]]
        if any(self.where[i] is not b for i in ids) or len({len(t) for t in toks}) != 1:
            raise ValueError("a step continues requests of one batch, all by the same number of tokens")
        if len(ids) != len(b.ids):  # the others wait: they keep rows of their own
            rest = b.split([i for i in b.ids if i not in set(ids)])
            for i in rest.ids:
                self.where[i] = rest
            b = b.split([i for i in b.ids if i in set(ids)])
            for i in b.ids:
                self.where[i] = b
        at = {i: r for r, i in enumerate(ids)}
        return b, torch.tensor([toks[at[i]] for i in b.ids], dtype=torch.long, device=device)

    @torch.no_grad()
    def step(self, entries: List[dict], end: List[str]) -> Optional[torch.Tensor]:
        """Run one step; fp32 logits [wanted, vocab] on the CPU, or None if nothing is wanted."""
        out = None
        if entries:
            V, device = self.model.cfg.vocab_size, self.model.embed.device
            ids, toks = [e["id"] for e in entries], [[int(t) for t in e["tokens"]] for e in entries]
            if len(set(ids)) != len(ids) or any(not t for t in toks):
                raise ValueError("an entry is listed twice or brings no token")
            if any(not 0 <= t < V for ts in toks for t in ts):
                raise ValueError("token id out of range")
            known = [i in self.where for i in ids]
            if any(known) and not all(known):
                raise ValueError("a step mixes new and live requests")
            b, inp = (self._go_on if all(known) else self._start)(ids, toks, device)
            h = self.model(inp, cache=b.cache)
            row, T = {i: r for r, i in enumerate(b.ids)}, inp.shape[1]
            rows = [row[e["id"]] for e in entries for _ in e.get("want", [])]
            cols = [T - len(t) + w for e, t in zip(entries, toks) for w in e.get("want", [])]
            if any(not 0 <= w < len(t) for e, t in zip(entries, toks) for w in e.get("want", [])):
                raise ValueError("a wanted place lies outside the entry's tokens")
            if rows:
                hw = h[torch.tensor(rows, device=device), torch.tensor(cols, device=device)]
                out = self.model.logits(hw).float().cpu()
            elif h.is_cuda:
                torch.cuda.synchronize()
        self._end(end)
        return out

    def _end(self, end: List[str]):
        gone = {i for i in end if i in self.where}
        for b in {id(self.where[i]): self.where[i] for i in gone}.values():
            keep = [i for i in b.ids if i not in gone]
            nb = b.split(keep) if keep else None
            for i in keep:
                self.where[i] = nb
        for i in gone:
            del self.where[i]


def parse_args(argv=None):
    p = argparse.ArgumentParser(prog="trace_run", description="Replay token ids step by step, write logits")
    p.add_argument("--model", required=True, help="folder with config.json and model.safetensors")
    p.add_argument("--dtype", choices=("bfloat16", "float32"), default="bfloat16")
    p.add_argument("--out", required=True, help="folder for <step>.f32")
    p.add_argument("--max-tokens", type=int, default=None, help="most tokens live requests hold at any time")
    p.add_argument("--device", default="cuda", help="torch device (cpu: the PyTorch forms of the ops)")
    return p.parse_args(argv)


def main(argv=None) -> int:
    a = parse_args(argv)
    device = torch.device(a.device)
    if device.type == "cuda":
        if not torch.cuda.is_available():
            raise RuntimeError("no GPU visible (pass --device cpu for the PyTorch forms of the ops)")
        os.environ["DLA_AUTOBUILD"] = "1"
    torch.backends.cuda.matmul.allow_tf32 = False
    torch.set_float32_matmul_precision("highest")
    bundle = load_causal_lm(a.model, gradient_checkpointing=False, device=device,
                            torch_dtype=getattr(torch, a.dtype))
    runner = TraceRunner(bundle.model.eval(), a.max_tokens)
    for line in sys.stdin:
        if not line.strip():
            continue
        d = json.loads(line)
        lg = runner.step(d.get("entries", []), d.get("end", []))
        if lg is not None:
            tmp = os.path.join(a.out, f".{d['step']}.f32")
            lg.contiguous().numpy().astype("<f4").tofile(tmp)
            os.replace(tmp, os.path.join(a.out, f"{d['step']}.f32"))
        print(f"done {d['step']}", flush=True)
    return 0


if __name__ == "__main__":
    sys.exit(main())
