"""Trace replay: given token ids through a language model, step by step, logits out.

A trace is a sequence of steps; a step brings the next tokens of some requests (portions of prompts beside single tokens, cut anywhere), names the
places whose logits are wanted, and lists the requests that end with it.  The replayer is a client of the serving path: requests with open
prompts go through ``MI355XARScheduler.feed`` / ``schedule`` and ``MI355XARWorker.execute_model`` like any others -- the same block pool,
state slots, batch and kernels; nothing is sampled.
"""
from __future__ import annotations

import argparse
import json
import os
import sys

import torch

from .payloads import SamplingParams
from .scheduler import Request
from .serving import serve

MAX_LIVE = 4           # requests live at a time: state slots of the engine
PAGE = 64              # callers count a request's tokens in units of this many (a multiple of the block size)


class Replayer:
    def __init__(self, model, dtype: str, max_tokens: int, *, max_live: int = MAX_LIVE, weights: dict | None = None, block_size: int = 16):
        """A cache pool for `max_tokens` tokens (and the null block), `max_live` state slots; nothing is sampled, so no graph is captured."""
        tokens = (max_tokens + PAGE - 1) // PAGE * PAGE
        self.core = serve(model, weights=weights, dtype=dtype, num_blocks=tokens // block_size + 1, block_size=block_size, max_num_seqs=max_live, max_model_len=tokens,
                          max_num_batched_tokens=tokens, enforce_eager=True)

    def step(self, entries: list[dict], end: list[str]) -> torch.Tensor | None:
        """entries: [{"id", "tokens", "want"}]; returns the wanted logits fp32 [wanted, vocab] in the order of the entries and of "want"."""
        sched = self.core.scheduler
        for e in entries:
            rid, tokens, want = e["id"], [int(t) for t in e["tokens"]], [int(k) for k in e.get("want") or ()]
            if not tokens or any(not 0 <= k < len(tokens) for k in want):
                raise ValueError(f"request {rid}: no tokens, or a wanted place outside them")
            if rid in sched.requests:
                sched.feed(rid, tokens, want)
            else:
                sched.add_request(Request(request_id=rid, num_prompt_tokens=len(tokens), prompt_token_ids=tokens, sampling_params=SamplingParams(temperature=0.0),
                                          open_prompt=True, logits_at=set(want)))
        so = sched.schedule()
        for e in entries:
            if so.num_scheduled_tokens.get(e["id"], 0) != len(e["tokens"]):
                raise RuntimeError(f"request {e['id']}: {so.num_scheduled_tokens.get(e['id'], 0)} of {len(e['tokens'])} tokens fit (cache pool or live requests exceeded)")
        out = self.core._dispatch(so)
        sched.update_from_output(so, out)
        rows = []
        for e in entries:
            want = [int(k) for k in e.get("want") or ()]
            if want:
                got, places = out.token_logits[e["id"]], so.logits_at[e["id"]]
                at = {k: j for j, k in enumerate(places)}
                rows.append(got[[at[k] for k in want]])
            if e["id"] in sched.requests:
                sched.requests[e["id"]].logits_at.clear()
        res = torch.cat(rows).float().cpu() if rows else None
        if res is None:
            torch.cuda.synchronize()
        for rid in end:
            sched.abort_request(rid)
        return res


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="trace_run", description="Feed given token ids through a language model, step by step (JSON steps on standard input), and "
                                 "write the wanted logits of every step to <out>/<step>.f32.")
    ap.add_argument("--model", required=True, help="directory with config.json and model.safetensors")
    ap.add_argument("--dtype", choices=("bfloat16", "float32"), default="bfloat16")
    ap.add_argument("--out", required=True, help="directory for the logits (little-endian fp32, [wanted, vocab])")
    ap.add_argument("--max-tokens", type=int, required=True, help="most tokens live requests hold at a time, each request rounded up to a multiple of 64")
    a = ap.parse_args(argv)
    os.makedirs(a.out, exist_ok=True)
    rep = Replayer(a.model, a.dtype, a.max_tokens)
    for line in sys.stdin:
        if not line.strip():
            continue
        s = json.loads(line)
        logits = rep.step(s.get("entries") or [], s.get("end") or [])
        if logits is not None:
            logits.contiguous().numpy().astype("<f4").tofile(os.path.join(a.out, f"{s['step']}.f32"))
        print(f"done {s['step']}", flush=True)
    return 0
