"""Decoder-only language models, everything that needs no GPU: configuration and registry, checkpoint checks, open prompts in the scheduler,
state slots, attention work items, and the oracle's mechanisms against loops over single numbers."""
import math

import pytest
import torch

from ht_vllm_omni_amd import models
from ht_vllm_omni_amd.checkpoint import load_decoder_checkpoint
from ht_vllm_omni_amd.config import TalkerDims
from ht_vllm_omni_amd.decoder_config import dims_from_config, tensor_shapes
from ht_vllm_omni_amd.decoder_engine import LATENT_WIDTHS, attention_tiles, latent_width
from ht_vllm_omni_amd.payloads import OmniModelRunnerOutput, SamplingParams
from ht_vllm_omni_amd.sched import SlotPool
from ht_vllm_omni_amd.scheduler import MI355XARScheduler, Request
from ht_vllm_omni_amd.worker import MI355XARWorker, make_config
from oracle import decoder_oracle as D
from tests.decoder_util import CONFIGS, G, config, layer, model


# ---------------------------------------------------------------- configuration
def test_config_gives_every_size_and_constant():
    cfg = config([layer(heads=7, dim=11, vdim=13, kv_rank=17, q_rank=19, scale=0.77, ff=23), layer(G, ff=None)], width=29, vocab=31, eps=3e-4)
    d = dims_from_config(cfg, 99)
    m = d.layers[0].mixer
    assert (m.heads, m.dim, m.vdim, m.kv_rank, m.q_rank, m.scale, m.out_gate) == (7, 11, 13, 17, 19, 0.77, False)
    assert d.layers[0].mlp.ff == 23 and d.layers[1].mlp is None and d.layers[1].mixer.out_gate
    assert (d.hidden, d.vocab, d.eps, d.max_model_len) == (29, 31, 3e-4, 99)


def test_borrowed_layers_have_no_tensors():
    d, w, cfg = model("mixed")
    assert [d.owner(i) for i in range(4)] == [0, 1, 0, 1]
    names = tensor_shapes(d)
    assert not any(n.startswith(("l2.", "l3.")) for n in names)
    assert "l0.mlp.up" in names and "l1.norm2" not in names and "l1.mix.g" in names and "l0.mix.g" not in names
    assert model("behind")[0].owner(0) == 1


@pytest.mark.parametrize("bad", [
    config([layer("sliding")]), config([dict(layer(), mlp={"kind": "experts", "ff": 8})]), config([layer(weights_of=3)]),
    config([layer(weights_of=1), layer(weights_of=0)]), config([layer(), layer(heads=2, weights_of=0)]), config([layer(heads=0)]),
    config([dict(layer(), mixer=dict(layer()["mixer"], window=8))])])
def test_unknown_or_contradictory_configs_are_refused(bad):
    with pytest.raises(ValueError):
        dims_from_config(bad)


def test_registry_tells_the_families_apart(tmp_path):
    assert models.entry_for_config(CONFIGS["mixed"]).name == "decoder"
    assert models.entry_for_config({"talker_config": {}}).name == "talker"
    assert models.entry_for_dims(model("mixed")[0]).name == "decoder"
    assert models.entry_for_dims_type(TalkerDims).name == "talker"
    with pytest.raises(ValueError):
        models.dims_of_model_dir({"architecture": "Another"})
    cfg = make_config(model("mixed")[0], max_num_seqs=3)
    assert cfg.kv_cache_dtype == "auto" and make_config("tiny").kv_cache_dtype == "fp8"
    spec = MI355XARWorker(cfg).get_kv_cache_spec()
    assert [s.width for s in spec.values()] == [64, 96, 64, 96] and MI355XARWorker(cfg).kv_bytes_per_block() == 16 * 2 * (64 + 96 + 64 + 96)
    assert MI355XARWorker(make_config(model("mixed")[0], dtype="float32")).kv_bytes_per_block() == 16 * 4 * (64 + 96 + 64 + 96)


def test_checkpoint_names_and_shapes_are_checked(tmp_path):
    from safetensors.torch import save_file
    d, w, _ = model("mixed")
    save_file(w, str(tmp_path / "model.safetensors"))
    got = load_decoder_checkpoint(str(tmp_path), d)
    assert set(got) == set(w) and all(torch.equal(got[k], w[k]) for k in w)
    for change in ({"l0.mix.uk": None}, {"l0.mix.uk": torch.zeros(2, 2)}, {"l9.mix.uk": torch.zeros(2, 2)}):
        v = {k: t for k, t in {**w, **change}.items() if t is not None}
        save_file(v, str(tmp_path / "model.safetensors"))
        with pytest.raises((KeyError, ValueError)):
            load_decoder_checkpoint(str(tmp_path), d)


# ---------------------------------------------------------------- scheduling
def _ran(so):
    ids = list(so.num_scheduled_tokens)
    return OmniModelRunnerOutput(ids, {r: i for i, r in enumerate(ids)}, [[] for _ in ids])


def test_open_prompts_are_fed_in_pieces_and_keep_their_blocks():
    s = MI355XARScheduler(num_blocks=9, block_size=4, max_num_seqs=2, max_num_batched_tokens=64, max_model_len=64)
    s.add_request(Request("a", 5, SamplingParams(), [1, 2, 3, 4, 5], open_prompt=True, logits_at={1, 4}))
    so = s.schedule()
    assert so.scheduled_new_reqs[0].open_prompt and so.num_scheduled_tokens == {"a": 5} and so.logits_at == {"a": [1, 4]}
    s.update_from_output(so, _ran(so))
    assert s.schedule().total_num_scheduled_tokens == 0                        # idle, not finished
    s.feed("a", [6, 7], logits_at=[1])
    s.add_request(Request("b", 2, SamplingParams(), [9, 9], open_prompt=True))
    so = s.schedule()
    c = so.scheduled_cached_reqs
    assert c.req_ids == ["a"] and c.new_token_ids == [[6, 7]] and so.num_scheduled_tokens == {"a": 2, "b": 2} and so.logits_at == {"a": [1]}
    s.update_from_output(so, _ran(so))
    assert s.pool.block_ids("a") == [1, 2] and s.pool.block_ids("b") == [3]
    s.abort_request("a")
    assert s.pool.num_free == 7 and s.schedule().finished_req_ids == {"a"}
    with pytest.raises(KeyError):
        s.feed("a", [1])


def test_a_fed_piece_larger_than_the_budget_runs_in_portions():
    s = MI355XARScheduler(num_blocks=9, block_size=4, max_num_seqs=2, max_num_batched_tokens=4, max_model_len=64)
    s.add_request(Request("a", 1, SamplingParams(), [1], open_prompt=True))
    so = s.schedule()
    s.update_from_output(so, _ran(so))
    s.feed("a", [2, 3, 4, 5, 6], logits_at=[0, 4])
    so = s.schedule()
    assert so.num_scheduled_tokens == {"a": 4} and so.scheduled_cached_reqs.new_token_ids == [[2, 3, 4, 5, 6]] and so.logits_at == {"a": [0]}
    s.update_from_output(so, _ran(so))
    so = s.schedule()
    assert so.num_scheduled_tokens == {"a": 1} and so.scheduled_cached_reqs.new_token_ids == [[]] and so.logits_at == {"a": [0]}


def test_state_slots_are_unique_and_come_back():
    p = SlotPool(3)
    got = [p.acquire(r) for r in "abc"]
    assert sorted(got) == [1, 2, 3]
    with pytest.raises(MemoryError):
        p.acquire("d")
    p.release("b")
    p.release("b")
    assert p.acquire("d") == got[1]


def test_attention_tiles_cover_every_row_once_and_never_straddle_sequences():
    for heads, rows in ((1, 64), (3, 128), (16, 64), (40, 128), (200, 64)):
        starts, lens = [2, 9, 140], [7, 131, 2]
        seen = []
        for f, n in attention_tiles(starts, lens, heads, rows):
            assert 1 <= n <= rows
            owner = [k for k, (s, c) in enumerate(zip(starts, lens)) if s * heads <= f and f + n <= (s + c) * heads]
            assert len(owner) == 1
            seen += range(f, f + n)
        assert sorted(seen) == list(range(2 * heads, 142 * heads))


def test_cache_rows_are_padded_to_widths_the_kernels_have():
    for r in range(1, 513):
        assert latent_width(r, 0) in LATENT_WIDTHS and r <= latent_width(r, 0) < r + 64 and latent_width(r, 1) == (r + 31) // 32 * 32
    assert latent_width(513, 0) == 544


# ---------------------------------------------------------------- the oracle's mechanisms, number by number
def test_oracle_norms_and_shift():
    x, g = torch.tensor([[1.0, -2.0, 3.0], [0.5, 0.0, -1.5]], dtype=torch.float64), torch.tensor(1.7, dtype=torch.float64)
    w, mu = torch.tensor([0.3, 2.0, -1.0], dtype=torch.float64), torch.tensor([0.0, 0.25, 1.0], dtype=torch.float64)
    for t in range(2):
        r = math.sqrt(sum(float(v) ** 2 for v in x[t]) / 3 + 0.01)
        for k in range(3):
            assert float(D.scalar_rms_norm(x, g, 0.01)[t, k]) == pytest.approx(float(x[t, k]) / r * 1.7)
            assert float(D.rms_norm(x, w, 0.01)[t, k]) == pytest.approx(float(x[t, k]) / r * float(w[k]))
            prev = float(x[t - 1, k]) if t else 0.0
            assert float(D.token_shift(x, mu)[t, k]) == pytest.approx(float(x[t, k]) + (prev - float(x[t, k])) * float(mu[k]))


def test_oracle_xielu():
    pq = torch.tensor([0.4, -1.3], dtype=torch.float64)
    z = torch.tensor([-30.0, -2.0, -1e-3, 0.0, 1e-3, 2.0, 30.0], dtype=torch.float64)
    sp = [math.log(1 + math.exp(float(v))) for v in pq]
    for v, got in zip(z.tolist(), D.xielu(z, pq).tolist()):
        want = sp[0] * v * v + v / 2 if v > 0 else (0.5 + sp[1]) * (math.exp(v) - 1 - v) + v / 2
        assert got == pytest.approx(want, abs=1e-12)


def test_oracle_attention_and_gate():
    g = torch.Generator().manual_seed(3)
    T, H, dim, vdim, W, R, Q = 5, 2, 3, 4, 6, 5, 7
    rnd = lambda *s: torch.randn(*s, generator=g, dtype=torch.float64)  # noqa: E731
    w = dict(dq=rnd(Q, W), dq_norm=rnd(Q), uq=rnd(H * dim, Q), dkv=rnd(R, W), dkv_norm=rnd(R), uk=rnd(H * dim, R), uv=rnd(H * vdim, R), o=rnd(W, H * vdim), g=rnd(H, W))
    h = rnd(T, W)
    for gated in (False, True):
        got = D.latent_attention(h, w, H, dim, vdim, 0.37, 1e-3, gated)
        rms = lambda v, n: v / math.sqrt(float((v * v).mean()) + 1e-3) * n  # noqa: E731
        for t in range(T):
            heads = []
            q = w["uq"] @ rms(w["dq"] @ h[t], w["dq_norm"])
            cs = [rms(w["dkv"] @ h[j], w["dkv_norm"]) for j in range(t + 1)]
            for n in range(H):
                s = [0.37 * float(q[n * dim:(n + 1) * dim] @ (w["uk"] @ c)[n * dim:(n + 1) * dim]) for c in cs]
                e = [math.exp(v - max(s)) for v in s]
                v = sum(a / sum(e) * (w["uv"] @ c)[n * vdim:(n + 1) * vdim] for a, c in zip(e, cs))
                heads.append(v * (1 / (1 + math.exp(-float(w["g"][n] @ h[t]))) if gated else 1.0))
            assert torch.allclose(got[t], w["o"] @ torch.cat(heads), atol=1e-10)


def test_oracle_borrowed_layer_is_the_owner_run_again():
    d, w, cfg = model("mixed")
    toks = [3, 1, 4, 1, 5]
    full = dict(cfg, layers=[dict(e, weights_of=None) for e in cfg["layers"]])
    copies = dict(w)
    for i, o in ((2, 0), (3, 1)):
        copies.update({k.replace(f"l{o}.", f"l{i}.", 1): t for k, t in w.items() if k.startswith(f"l{o}.")})
    assert torch.equal(D.zefedra_forward(w, cfg, toks)[0], D.zefedra_forward(copies, full, toks)[0])
