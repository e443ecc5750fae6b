"""Command line: ``python -m ht_vllm_omni_amd generate`` (token ids in, token ids out, through worker and scheduler) and ``trace`` (bin/trace_run)."""
from __future__ import annotations

import argparse
import json
import sys


def generate(argv) -> int:
    ap = argparse.ArgumentParser(prog="generate", description="Generate from token-id prompts with a decoder-only language model.")
    ap.add_argument("--model", required=True, help="directory with config.json and model.safetensors")
    ap.add_argument("--dtype", choices=("bfloat16", "float32"), default="bfloat16")
    ap.add_argument("--prompt", action="append", required=True, help="comma-separated token ids (repeat for more requests)")
    ap.add_argument("--max-tokens", type=int, default=16)
    ap.add_argument("--temperature", type=float, default=0.0, help="0: greedy")
    ap.add_argument("--top-k", type=int, default=0)
    ap.add_argument("--top-p", type=float, default=1.0)
    ap.add_argument("--seed", type=int, default=None)
    ap.add_argument("--max-model-len", type=int, default=4096)
    ap.add_argument("--max-num-seqs", type=int, default=64)
    ap.add_argument("--max-num-batched-tokens", type=int, default=8192)
    ap.add_argument("--num-blocks", type=int, default=None, help="cache blocks of 16 tokens (default: what the prompts need)")
    a = ap.parse_args(argv)
    from .build import ensure_decoder
    from .payloads import SamplingParams
    from .scheduler import Request
    from .serving import serve
    ensure_decoder()
    prompts = [[int(t) for t in p.split(",")] for p in a.prompt]
    need = sum((len(p) + a.max_tokens + 15) // 16 for p in prompts) + 1
    core = serve(a.model, dtype=a.dtype, num_blocks=a.num_blocks or need, max_num_seqs=a.max_num_seqs, max_model_len=a.max_model_len,
                 max_num_batched_tokens=a.max_num_batched_tokens)
    sp = SamplingParams(temperature=a.temperature, top_k=a.top_k, top_p=a.top_p, repetition_penalty=1.0, seed=a.seed, max_tokens=a.max_tokens, stop_token_ids=())
    for i, p in enumerate(prompts):
        core.add_request(Request(request_id=str(i), num_prompt_tokens=len(p), prompt_token_ids=p, sampling_params=sp))
    out = core.run()
    for i in range(len(prompts)):
        print(json.dumps({"request": i, "token_ids": out.get(str(i), [])}))
    return 0


def main() -> int:
    cmd = sys.argv[1] if len(sys.argv) > 1 else ""
    if cmd == "generate":
        return generate(sys.argv[2:])
    if cmd == "trace":
        from .build import ensure_decoder
        ensure_decoder()
        from .replay import main as trace
        return trace(sys.argv[2:])
    print("usage: python -m ht_vllm_omni_amd {generate,trace} ...", file=sys.stderr)
    return 2


if __name__ == "__main__":
    sys.exit(main())
