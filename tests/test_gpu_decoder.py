"""Decoder-only language models end to end on the GPU, against the plain whole-sequence oracle: prompts, decoding, portions, mixed batches, reused
pages and slots, generation through scheduler and runner, the command line."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

from ht_vllm_omni_amd.decoder_engine import DecoderEngine
from ht_vllm_omni_amd.payloads import SamplingParams
from ht_vllm_omni_amd.replay import Replayer
from ht_vllm_omni_amd.scheduler import Request
from ht_vllm_omni_amd.serving import serve
from tests.decoder_util import CONFIGS, TOL, assert_logits, model, oracle, oracle_logits, tokens

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
DTYPES = ["float32", "bfloat16"]


def feed(rep, rid, toks, cuts, end=True):
    """One request alone in portions of the given sizes (the last size repeats); logits of every token."""
    out, o, i = [], 0, 0
    while o < len(toks):
        n = min(cuts[min(i, len(cuts) - 1)], len(toks) - o)
        last = o + n == len(toks)
        out.append(rep.step([{"id": rid, "tokens": toks[o:o + n], "want": list(range(n))}], [rid] if last and end else []))
        o, i = o + n, i + 1
    return torch.cat(out)


# ---------------------------------------------------------------- layers, prompts
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(CONFIGS))
def test_residual_stream_of_every_layer(name, dtype):
    d, w, cfg = model(name, seed=1)
    eng = DecoderEngine(d, w, dtype=dtype, num_blocks=20, max_batch=3, block_size=8)
    eng.block_table[2, :10] = torch.randperm(19, device="cuda")[:10].to(torch.int32) + 1
    eng.state_slot[2] = 3
    toks = tokens(77, d.vocab)
    b = eng.make_batch(torch.tensor(toks), np.full(77, 2), np.arange(77), [77])
    trail = []
    logits = eng.forward(b, trail=trail)
    ref, ref_trail = oracle(w, cfg, toks)
    for i, (a, r) in enumerate(zip(trail, ref_trail)):
        err = float((a.cpu() - r).pow(2).mean().sqrt() / r.pow(2).mean().sqrt())
        assert err <= TOL[dtype], f"layer {i}: {err:.3g}"
    assert len(trail) == d.num_layers
    assert_logits(logits[:, :d.vocab], ref, dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("n", [1, 2, 16, 17, 64, 65, 300, 700])
@pytest.mark.parametrize("name", ["mixed", "k_mixed"])
def test_whole_prompts(name, n, dtype):
    d, w, cfg = model(name, seed=2, sharp=3.0)
    rep = Replayer(d, dtype, 1024, weights=w)
    toks = tokens(n, d.vocab, n)
    assert_logits(feed(rep, "a", toks, [n]), oracle_logits(w, cfg, toks), dtype, f"{n} tokens")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["wide", "k_wide", "k_plain"])
def test_wide_model_long_prompt(name, dtype):
    d, w, cfg = model(name, seed=3, sharp=2.0)
    rep = Replayer(d, dtype, 1024, weights=w)
    toks = tokens(600, d.vocab, 5)
    assert_logits(feed(rep, "a", toks, [590, 1]), oracle_logits(w, cfg, toks), dtype)


# ---------------------------------------------------------------- decoding and portions
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["mixed", "narrow", "behind", "k_mixed", "k_narrow", "k_state"])
def test_token_by_token_equals_the_whole_prompt(name, dtype):
    d, w, cfg = model(name, seed=4, sharp=4.0)
    rep = Replayer(d, dtype, 128, weights=w)
    toks = tokens(70, d.vocab, 6)
    one = feed(rep, "a", toks, [1])
    assert_logits(one, oracle_logits(w, cfg, toks), dtype)
    assert_logits(feed(rep, "b", toks, [70]), one.float(), dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("cuts", [[2], [3, 2], [16], [15, 2, 31, 1, 1, 5], [64, 2], [65, 64], [33, 1]])
@pytest.mark.parametrize("name", ["mixed", "k_mixed", "k_wide"])
def test_portions(name, cuts, dtype):
    d, w, cfg = model(name, seed=5, sharp=4.0)
    rep = Replayer(d, dtype, 256, weights=w)
    toks = tokens(190, d.vocab, 7)
    assert_logits(feed(rep, "a", toks, cuts), oracle_logits(w, cfg, toks), dtype, str(cuts))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name,sharp", [("narrow", 8.0), ("k_mixed", 3.0)])
def test_long_decoding_with_far_keys(name, sharp, dtype):
    """Sharp scores (single keys decide), 400 decoded tokens behind a prompt of 3: keys hundreds of tokens back, over many page borders."""
    d, w, cfg = model(name, seed=6, sharp=sharp)
    rep = Replayer(d, dtype, 512, weights=w)
    toks = tokens(403, d.vocab, 8)
    assert_logits(feed(rep, "a", toks, [3, 1]), oracle_logits(w, cfg, toks), dtype)


# ---------------------------------------------------------------- batches, pages, slots
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["mixed", "wide", "k_mixed", "k_wide", "k_plain", "k_state"])
def test_mixed_batches_equal_each_request_alone(name, dtype):
    """Up to four live requests at different places, portions beside single tokens, some left out of a step, ends and re-admissions into a pool
    that only just holds them: pages and slots change owners all the time."""
    d, w, cfg = model(name, seed=7, sharp=3.0)
    rep = Replayer(d, dtype, 448, weights=w)
    g = torch.Generator().manual_seed(9)
    lens = [130, 3, 61, 95, 1, 90, 40, 17, 66, 2]
    reqs = {f"r{i}": tokens(n, d.vocab, 20 + i) for i, n in enumerate(lens)}
    refs = {k: oracle_logits(w, cfg, t) for k, t in reqs.items()}
    waiting, live, got = list(reqs), {}, {k: [] for k in reqs}
    room = lambda: 448 - sum(-(-len(reqs[k]) // 64) * 64 for k in live)  # noqa: E731
    seen_mixed = 0
    while waiting or live:
        while waiting and len(live) < 4 and -(-len(reqs[waiting[0]]) // 64) * 64 <= room():
            live[waiting.pop(0)] = 0
        entries, end = [], []
        for k in sorted(live, key=lambda _: float(torch.rand((), generator=g))):
            if float(torch.rand((), generator=g)) < 0.2 and len(live) > 1:
                continue                                                # left out of this step
            n = [1, 1, 2, 5, 16, 37][int(torch.randint(0, 6, (), generator=g))]
            n = min(n, len(reqs[k]) - live[k])
            entries.append({"id": k, "tokens": reqs[k][live[k]:live[k] + n], "want": list(range(n))})
            if live[k] + n == len(reqs[k]):
                end.append(k)
        if not entries:
            continue
        sizes = [len(e["tokens"]) for e in entries]
        seen_mixed += 1 in sizes and max(sizes) > 1
        out = rep.step(entries, end)
        o = 0
        for e in entries:
            n = len(e["tokens"])
            got[e["id"]].append(out[o:o + n])
            o += n
            live[e["id"]] += n
        for k in end:
            del live[k]
    assert seen_mixed >= 5
    for k in reqs:
        assert_logits(torch.cat(got[k]), refs[k], dtype, k)


@pytest.mark.parametrize("name", ["mixed", "k_mixed"])
def test_a_reused_slot_and_page_hold_nothing_of_their_last_owner(name):
    """The same request before and after the pool was filled by others: identical bits."""
    d, w, _ = model(name, seed=8)
    rep = Replayer(d, "bfloat16", 128, max_live=1, weights=w)
    toks = tokens(50, d.vocab, 3)
    first = feed(rep, "a", toks, [20, 1])
    for i in range(3):
        feed(rep, f"x{i}", tokens(120, d.vocab, 40 + i), [120])
    assert torch.equal(feed(rep, "b", toks, [20, 1]), first)


def test_wanted_places_come_back_in_the_order_asked():
    d, w, cfg = model("narrow", seed=9)
    rep = Replayer(d, "float32", 256, weights=w)
    a, b = tokens(9, d.vocab, 1), tokens(30, d.vocab, 2)
    ra, rb = oracle_logits(w, cfg, a), oracle_logits(w, cfg, b)
    assert rep.step([{"id": "a", "tokens": a[:4], "want": []}], []) is None
    out = rep.step([{"id": "b", "tokens": b, "want": [29, 0, 7]}, {"id": "a", "tokens": a[4:], "want": [4, 1]}], ["a"])
    assert_logits(out, torch.stack([rb[29], rb[0], rb[7], ra[8], ra[5]]), "float32")
    with pytest.raises(RuntimeError, match="pool|fit"):
        rep.step([{"id": "c", "tokens": [1] * 250, "want": []}], [])


# ---------------------------------------------------------------- generation: scheduler, runner, sampler, graphs
def greedy_oracle(w, cfg, prompt, n, dtype=torch.float64):
    toks, margins = list(prompt), []
    for _ in range(n):
        top = torch.topk(oracle_logits(w, cfg, toks, dtype)[-1], 2)
        margins.append(float(top.values[0] - top.values[1]))
        toks.append(int(top.indices[0]))
    return toks[len(prompt):], margins


def generate(d, w, prompts, n, **kw):
    sp = kw.pop("sampling", None) or SamplingParams(temperature=0.0, repetition_penalty=1.0, max_tokens=n, stop_token_ids=())
    core = serve(d, weights=w, **kw)
    for i, p in enumerate(prompts):
        core.add_request(Request(str(i), len(p), sp, list(p)))
    out = core.run()
    return [out[str(i)] for i in range(len(prompts))], core


@pytest.mark.parametrize("name", ["mixed", "wide", "k_mixed", "k_narrow"])
def test_greedy_generation_equals_the_oracles(name):
    """fp32 through the engine-core loop: prompts that chunk over the token budget, decode graphs, requests that finish and make room."""
    d, w, cfg = model(name, seed=10, sharp=2.0)
    prompts = [tokens(n, d.vocab, 60 + n) for n in (1, 5, 40, 23, 16, 2)]
    got, core = generate(d, w, prompts, 12, dtype="float32", num_blocks=40, max_num_seqs=3, max_num_batched_tokens=24, max_model_len=64)
    assert core.worker.model_runner.cudagraph_stats["replays"] > 0
    for p, g in zip(prompts, got):
        want, margins = greedy_oracle(w, cfg, p, 12)
        assert g == want or min(margins) < 1e-4, (g, want, min(margins))


@pytest.mark.parametrize("name", ["mixed", "k_mixed"])
def test_generation_does_not_depend_on_how_it_is_run(name):
    """bf16: graphs or eager, synchronous or asynchronous, ample or scarce cache (preemption: recomputed requests), seeded sampling -- the same ids
    up to near-ties, and the same ids exactly where the kernels are the same."""
    d, w, _ = model(name, seed=11)
    prompts = [tokens(n, d.vocab, 80 + n) for n in (7, 30, 18, 25)]
    sp = SamplingParams(temperature=0.8, top_k=20, repetition_penalty=1.1, seed=5, max_tokens=20, stop_token_ids=(), logprobs=2)
    base = dict(num_blocks=40, max_num_seqs=4, max_model_len=128, sampling=sp)
    ref, _ = generate(d, w, prompts, 20, **base)
    assert all(len(r) == 20 for r in ref)
    assert generate(d, w, prompts, 20, enforce_eager=True, **base)[0] == ref
    assert generate(d, w, prompts, 20, async_scheduling=True, **base)[0] == ref
    tight, core = generate(d, w, prompts, 20, dtype="float32", **dict(base, num_blocks=9))
    roomy, _ = generate(d, w, prompts, 20, dtype="float32", **base)
    assert tight == roomy, "preempted requests must carry on where they were"


@pytest.mark.parametrize("name", ["behind", "k_mixed"])
def test_replays_of_a_captured_step_match_eager_steps(name):
    """A captured decode step replayed several times, with the runner's own eager prompt steps between the replays, against an engine that never
    captures (same bits: same kernels)."""
    d, w, _ = model(name, seed=12)
    outs = []
    for eager in (False, True):
        sp = SamplingParams(temperature=0.0, repetition_penalty=1.0, max_tokens=9, stop_token_ids=())
        core = serve(d, weights=w, num_blocks=60, max_num_seqs=3, max_model_len=64, enforce_eager=eager)
        toks = {}
        for i in range(7):                              # one new request every other step: prompt steps between decode steps
            core.add_request(Request(str(i), 4 + i, sp, tokens(4 + i, d.vocab, i)))
            for _ in range(2):
                for o in core.step():
                    toks.setdefault(o.request_id, []).extend(o.new_token_ids)
        for k, v in core.run().items():
            toks.setdefault(k, []).extend(v)
        stats = core.worker.model_runner.cudagraph_stats
        assert (stats["replays"] == 0) == eager
        outs.append(toks)
    assert outs[0] == outs[1] and all(len(v) == 9 for v in outs[0].values())


def test_stops_logprobs_and_seeds():
    d, w, cfg = model("narrow", seed=13)
    p = tokens(6, d.vocab, 1)
    want, margins = greedy_oracle(w, cfg, p, 8)
    assert min(margins) > 1e-4
    stop = want[4]
    core = serve(d, weights=w, dtype="float32", num_blocks=20, max_num_seqs=2, max_model_len=64)
    core.add_request(Request("a", 6, SamplingParams(temperature=0.0, repetition_penalty=1.0, max_tokens=50, stop_token_ids=(stop,), logprobs=1), p))
    outs = []
    while core.has_work():
        outs += core.step()
    ids = [t for o in outs for t in o.new_token_ids]
    assert ids == want[:want.index(stop) + 1] and outs[-1].finish_reason == "stop"
    lg = oracle_logits(w, cfg, p)[-1]
    lp = outs[0].new_logprobs
    assert lp.logprob_token_ids[0][0] == ids[0] and abs(lp.logprobs[0][0] - float(torch.log_softmax(lg, -1)[ids[0]])) < 1e-4
    assert core.scheduler.pool.num_free == 19 and not core.worker.model_runner.slots.owned


@pytest.mark.parametrize("name", ["mixed", "k_mixed"])
def test_worker_measures_memory_and_resizes_the_cache(name):
    d, w, cfg = model(name, seed=14)
    from ht_vllm_omni_amd.worker import MI355XARWorker, make_config
    wk = MI355XARWorker(make_config(d.with_(max_model_len=256), weights=w, max_num_seqs=2))
    wk.init_device()
    wk.load_model()
    wk.vllm_config.max_num_batched_tokens = 512
    wk.vllm_config.kv_cache_memory_bytes = 24 * wk.kv_bytes_per_block()
    wk.initialize_from_config(None)
    assert wk.engine.num_blocks == 24 and wk.engine.kv_cache_bytes() == 24 * wk.kv_bytes_per_block()


# ---------------------------------------------------------------- command line
@pytest.mark.parametrize("name", ["behind", "k_narrow"])
def test_command_lines(name, tmp_path):
    """bin/trace_run and `generate` on a checkpoint directory, in processes of their own."""
    from safetensors.torch import save_file
    d, w, cfg = model(name, seed=15)
    save_file(w, str(tmp_path / "model.safetensors"))
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    toks = tokens(21, d.vocab, 4)
    ref = oracle_logits(w, cfg, toks)
    steps = [{"step": 0, "entries": [{"id": "q", "tokens": toks[:18], "want": [0, 17]}], "end": []},
             {"step": 1, "entries": [{"id": "q", "tokens": toks[18:20], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "q", "tokens": toks[20:], "want": [0]}], "end": ["q"]}]
    out = tmp_path / "out"
    r = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", str(tmp_path), "--dtype", "float32", "--out", str(out), "--max-tokens", "64"],
                       input="\n".join(json.dumps(s) for s in steps), capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [ln for ln in r.stdout.split("\n") if ln.startswith("done")] == ["done 0", "done 1", "done 2"]
    assert sorted(os.listdir(out)) == ["0.f32", "2.f32"]
    got = np.concatenate([np.fromfile(out / f, dtype="<f4").reshape(-1, d.vocab) for f in ("0.f32", "2.f32")])
    assert_logits(torch.from_numpy(got), ref[[0, 17, 20]], "float32")
    r = subprocess.run([sys.executable, "-m", "ht_vllm_omni_amd", "generate", "--model", str(tmp_path), "--dtype", "float32", "--prompt", ",".join(map(str, toks)),
                        "--max-tokens", "5"], capture_output=True, text=True, timeout=100, cwd=ROOT)
    assert r.returncode == 0, r.stderr[-2000:]
    want, margins = greedy_oracle(w, cfg, toks, 5)
    assert min(margins) > 1e-4 and json.loads(r.stdout.strip().split("\n")[-1])["token_ids"] == want


@pytest.mark.parametrize("name", ["mixed", "k_mixed"])
def test_an_engine_out_of_use_gives_its_memory_back_at_once(name):
    """No reference circle keeps it for the collector: the next engine's memory accounting would count it."""
    import gc
    import weakref
    d, w, _ = model(name, seed=16)
    gc.collect()
    gc.disable()
    try:
        eng = DecoderEngine(d, w, num_blocks=8, max_batch=2)
        gone = weakref.ref(eng)
        eng.forward(eng.make_batch(torch.tensor([1, 2, 3]), [0] * 3, [0, 1, 2], [3]))
        del eng
        assert gone() is None
    finally:
        gc.enable()
