"""Trace replay: given token ids through a model's step function, logits to files.

    bin/trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N

Standard input holds one JSON step per line:

    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": []}

The entries of a step are one batch of the engine's runner: each continues its request by ``tokens`` (portions
of prompts and single tokens mixed; a request takes a slot at its first entry and may skip steps). ``want``
lists places among the tokens whose logits are wanted; they go to DIR/<step>.f32 (little-endian fp32,
[wanted, vocab], in the order of the entries). ``end`` names requests whose slot and pages are given back after
the step. ``done <step>`` on standard output closes every step. The cache pool holds N tokens (rounded up to
whole pages) and ``SLOTS`` requests.
"""
from __future__ import annotations

import argparse
import json
import os
import sys

SLOTS = 4
DTYPES = ("bfloat16", "float32")


class Replay:
    """Request ids on top of a runner's slots."""

    def __init__(self, runner):
        self.runner = runner
        self.free = list(range(runner.max_slots))[::-1]
        self.live: dict = {}  # id -> [slot, tokens so far]

    def step(self, entries, end):
        """-> logits of the wanted places (fp32, host) or None."""
        batch = []
        for e in entries:
            if e["id"] not in self.live:
                if not self.free:
                    raise RuntimeError(f"request {e['id']!r}: all {self.runner.max_slots} slots are taken")
                self.live[e["id"]] = [self.free.pop(), 0]
            slot, n = self.live[e["id"]]
            batch.append((slot, e["tokens"], n, e["want"]))
            self.live[e["id"]][1] += len(e["tokens"])
        logits = self.runner.forward_tokens(batch) if batch else None
        out = None if logits is None else logits.float().cpu()
        for i in end:
            slot, _ = self.live.pop(i)
            self.runner.release(slot)
            self.free.append(slot)
        return out


def open_runner(model_dir: str, dtype, max_tokens: int, device):
    """The serving runner of a model directory, with a page pool of ``max_tokens``."""
    from ..io.hf import load_pretrained
    from ..models.registry import family_of
    model = load_pretrained(model_dir, device=device, dtype=dtype)
    cls = family_of(model.cfg).runner()
    if not cls.mixed_steps:
        raise SystemExit(f"{model.cfg.arch}: this family's runner has no mixed steps")
    page = cls.default_page_size()
    pages = -(-max_tokens // page)
    return cls(model, max_slots=SLOTS, max_len=pages * page, use_graphs=False, page_size=page, kv_pages=pages)


def replay(runner, lines, out_dir: str, say):
    rp = Replay(runner)
    for line in lines:
        if not line.strip():
            continue
        s = json.loads(line)
        logits = rp.step(s["entries"], s["end"])
        if logits is not None:
            path = os.path.join(out_dir, f"{s['step']}.f32")
            with open(path + ".part", "wb") as f:
                f.write(logits.contiguous().numpy().astype("<f4", copy=False).tobytes())
            os.replace(path + ".part", path)
        say(f"done {s['step']}")


def main(argv=None):
    ap = argparse.ArgumentParser(description="Replay a trace of token ids and write the wanted logits")
    ap.add_argument("--model", required=True, help="model directory (config.json, model.safetensors)")
    ap.add_argument("--dtype", choices=DTYPES, required=True)
    ap.add_argument("--out", required=True, help="folder of the logits files")
    ap.add_argument("--max-tokens", type=int, required=True, help="tokens the cache pool holds")
    a = ap.parse_args(argv)
    import torch

    from ..models.registry import family_of_dict, read_dict
    from ..ops import _lib
    if not torch.cuda.is_available():
        raise SystemExit("no GPU: the kernels run on gfx950")
    _lib.ensure_built(family_of_dict(read_dict(a.model)).kernels)
    torch.set_float32_matmul_precision("highest")
    dev = torch.device("cuda", 0)
    runner = open_runner(a.model, getattr(torch, a.dtype), a.max_tokens, dev)
    replay(runner, sys.stdin, a.out, lambda t: print(t, flush=True))


if __name__ == "__main__":
    main()
