"""Replay a trace: token ids through a model step by step, logits out, nothing sampled.

    bin/trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N  < steps

Every input line is one step, {"step": n, "entries": [{"id": .., "tokens": [..], "want": [places in tokens]}, ..], "end": [ids]}; a step's
entries are one batch.  Requests that start together are prefilled as one left-padded batch (processor.collate_requests) and then
advance together, one token each, through the captured greedy step that generation replays -- with the trace's token in place of the
sampled one.  A request that ends leaves its batch row idle (every key masked); the batch's cache goes with its last request.  For a
step that wants logits, OUT/<step>.f32 holds them as little-endian float32 [wanted, vocab]; 'done <step>' is printed after every step.
"""
import argparse
import json
import os
import sys

import numpy as np


class Batch:
    """Requests that started together: their rows of one cache."""

    def __init__(self, model, entries, max_tokens):
        from .processor import collate_requests
        lens = [len(e["tokens"]) for e in entries]
        reqs = [{"input_ids": np.asarray(e["tokens"], dtype=np.int64)[None]} for e in entries]
        inputs = collate_requests(reqs) if len(reqs) > 1 else reqs[0]
        self.model, self.row = model, {e["id"]: i for i, e in enumerate(entries)}
        # a live request holds at most max_tokens tokens, so no row advances further than that behind its own prompt
        room = max(1, max_tokens - min(lens))
        logits, self.cache = model(**inputs, max_tokens=room, full_logits=True)
        self.tokens = [0] * len(lens)
        self.pads = [max(lens) - n for n in lens]
        self.logits = logits                                     # [rows, longest prompt, vocab]

    def advance(self, entries):
        """One token for each of `entries`; returns logits [rows, 1, vocab]."""
        import torch
        tok = list(self.tokens)
        for e in entries:
            tok[self.row[e["id"]]] = e["tokens"][0]
        logits, _ = self.model.greedy_step(torch.tensor(tok, dtype=torch.int32, device=self.model.device).view(-1, 1), self.cache)
        self.logits, self.pads = logits, [0] * len(tok)

    def wanted(self, entry):
        """Row of the last step's logits for every wanted place."""
        r = self.row[entry["id"]]
        return [self.logits[r, self.pads[r] + w] for w in entry["want"]]

    def end(self, rid):
        """The request is over: its row's keys are masked from now on."""
        import torch
        st, r = self.cache[0].state, self.row.pop(rid)
        if not self.row:
            return
        if st.pad_len is None:                                   # (captured steps bake the pointer in: none has been captured without it)
            st.graphs.clear()
            st.pad_len = torch.zeros((st.B,), dtype=torch.int32, device=self.model.device)
        st.pad_len[r:r + 1].fill_(st.Tp)


class Replay:
    def __init__(self, model, max_tokens):
        self.model, self.max_tokens, self.of = model, max_tokens, {}

    def step(self, entries):
        """Run one step's entries; returns their wanted logits in order, as a list of rows."""
        fresh = [e for e in entries if e["id"] not in self.of]
        touched = []
        if fresh:
            b = Batch(self.model, fresh, self.max_tokens)
            self.of.update((e["id"], b) for e in fresh)
            touched.append((b, fresh))
        going = {}
        for e in entries:
            if not any(e is f for f in fresh):
                if len(e["tokens"]) != 1:
                    raise ValueError(f"request {e['id']!r} goes on by {len(e['tokens'])} tokens; a started request advances by one")
                going.setdefault(id(self.of[e["id"]]), []).append(e)
        for es in going.values():
            b = self.of[es[0]["id"]]
            if len(es) != len(b.row):
                raise ValueError("the live requests of a batch advance together")
            b.advance(es)
            touched.append((b, es))
        rows = {id(e): b.wanted(e) for b, es in touched for e in es if e["want"]}
        return [r for e in entries for r in rows.get(id(e), [])]

    def end(self, ids):
        for rid in ids:
            b = self.of.pop(rid, None)
            if b is not None:
                b.end(rid)


def main(argv=None):
    ap = argparse.ArgumentParser(prog="trace_run", description="replay a trace of token ids through a model, step by step")
    ap.add_argument("--model", required=True, help="folder with config.json and model.safetensors")
    ap.add_argument("--dtype", default="bfloat16", choices=("bfloat16", "float32"))
    ap.add_argument("--out", required=True, help="folder for <step>.f32")
    ap.add_argument("--max-tokens", type=int, default=4096, help="most tokens that live requests hold at any time")
    a = ap.parse_args(argv)
    import torch
    from . import _lib
    from .api import load
    from .config import load_config
    from .registry import family
    units = family(load_config(os.path.join(a.model, "config.json"))).units
    if units:
        _lib.build_units(units)
    model, _ = load(model_path=a.model, dtype=a.dtype)
    replay = Replay(model, a.max_tokens)
    for line in sys.stdin:
        if not line.strip():
            continue
        s = json.loads(line)
        rows = replay.step(s["entries"])
        if rows:
            torch.stack(rows).float().cpu().numpy().astype("<f4").tofile(os.path.join(a.out, f"{s['step']}.f32"))
        replay.end(s.get("end", []))
        print(f"done {s['step']}", flush=True)
    return 0


if __name__ == "__main__":
    sys.exit(main())
