"""Decoder-only language models, everything that needs no GPU: configuration and registry, checkpoint checks, open prompts in the scheduler,
state slots, attention work items, and the oracle's mechanisms against loops over single numbers."""
import math

import pytest
import torch

from ht_vllm_omni_amd import models
from ht_vllm_omni_amd.checkpoint import load_decoder_checkpoint
from ht_vllm_omni_amd.config import TalkerDims
from ht_vllm_omni_amd.decoder_config import dims_from_config, tensor_shapes
from ht_vllm_omni_amd.decoder_mixers import (LATENT_WIDTHS, attention_tiles, cache_row_widths, cache_traffic, latent_width, pad_head_cols, pad_head_rows, pad_heads,
                                             recurrence_chunks, recurrence_segments, state_bytes)
from ht_vllm_omni_amd.payloads import OmniModelRunnerOutput, SamplingParams
from ht_vllm_omni_amd.sched import SlotPool
from ht_vllm_omni_amd.scheduler import MI355XARScheduler, Request
from ht_vllm_omni_amd.worker import MI355XARWorker, make_config
from oracle import decoder_oracle as D
from tests.decoder_util import CONFIGS, G, attention, config, koronex, layer, lightning, model


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


# ---------------------------------------------------------------- Koronex
def test_koronex_config_gives_every_size_and_constant():
    cfg = koronex([lightning(3, 11, 13, [0.25, 0.5, 1.0], ff=None), attention(6, 3, 14, 9, 0.77, 5, 6, 321.0, ff=23), attention(2, 3 - 2, 4, 5, 0.1, 7, 0, 2.0),
                   attention(9, 3, 14, 9, 0.5, 2, 6, 321.0, kv_from=1)], width=29, vocab=31, eps=3e-4, alpha=1.25, scale=0.5, side=7)
    d = dims_from_config(cfg, 99)
    a, b = d.layers[0].mixer, d.layers[1].mixer
    assert (a.heads, a.dim, a.vdim, a.decay) == (3, 11, 13, (0.25, 0.5, 1.0)) and d.layers[0].mlp is None
    assert (b.heads, b.kv_heads, b.dim, b.vdim, b.scale, b.window, b.rot_dims, b.rot_base, b.kv_from) == (6, 3, 14, 9, 0.77, 5, 6, 321.0, None)
    assert b.qk_norm and b.sink and b.out_gate and (d.layers[1].mlp.ff, d.layers[1].mlp.act) == (23, "relu2")
    assert (d.layers[3].mixer.kv_from, d.layers[3].mixer.window, d.kv_owner(3), d.kv_owner(1), d.kv_owner(0)) == (1, 2, 1, 1, None)
    assert (d.hidden, d.vocab, d.eps, d.alpha, d.embed_scale, d.side_dim, d.norm, d.token_shift, d.max_model_len) == (29, 31, 3e-4, 1.25, 0.5, 7, "post", False, 99)
    names = tensor_shapes(d)
    assert names["side.embed"] == (31, 4 * 7) and names["l0.mix.norm"] == (3 * 13,) and names["l1.mix.k.norm"] == (3 * 14,) and names["l3.mix.q.norm"] == (9 * 14,)
    assert names["l1.mix.g"] == (6 * 9, 29) and names["l1.mix.sink"] == (6,) and names["final.norm"] == (29,) and names["l2.side.proj"] == (29, 7)
    assert not any(n.startswith("l3.mix.") and n.split(".")[2] in ("k", "v") for n in names) and "l0.norm2" not in names and "l1.shift" not in names


@pytest.mark.parametrize("layers", [
    [attention(kv_from=0)], [attention(), attention(kv_from=1)], [lightning(), attention(kv_from=0)], [attention(), attention(kv_from=0), attention(kv_from=1)],
    [attention(), attention(kv_from=0, dim=44)], [attention(), attention(kv_from=0, rot=8)], [attention(), attention(3, 1, kv_from=0)], [attention(7, 2)], [attention(rot=41)],
    [attention(rot=42)], [attention(window=0)], [lightning(2, decay=[0.5])], [lightning(1, decay=[0.0])], [dict(lightning(), type="delta")], [dict(attention(), weights_of=0)],
    [dict(attention(), mlp={"kind": "experts", "ff": 8})], [dict(attention(), mixer=dict(attention()["mixer"], cap=30.0))],
    [dict(attention(), mixer={k: v for k, v in attention()["mixer"].items() if k != "rot"})]])
def test_unknown_or_contradictory_koronex_configs_are_refused(layers):
    with pytest.raises(ValueError):
        dims_from_config(koronex(layers))


def test_what_a_layer_keeps():
    """Cache pages for layers with keys of their own, state for recurrences, neither for a layer that reads another's."""
    d = model("k_mixed")[0]
    assert models.entry_for_dims(d).name == "decoder" and models.entry_for_config(CONFIGS["k_mixed"]).name == "decoder"
    assert [sum(cache_row_widths(d, i, 0)) for i in range(6)] == [2 * (64 + 32), 0, 0, 0, 4 * 64, 0]
    wk = MI355XARWorker(make_config(d, max_num_seqs=3))
    assert sorted(wk.get_kv_cache_spec()) == ["model.layers.0.mixer", "model.layers.4.mixer"] and wk.kv_bytes_per_block() == 16 * 2 * (192 + 256)
    assert [state_bytes(d, i) for i in range(6)] == [0, 4 * 3 * 24 * 40, 0, 4 * 2 * 40 * 16, 0, 0]
    assert cache_traffic(d, 2, 100) == (20 * 2 * 64, 0) and cache_traffic(d, 0, 4) == (4 * 2 * 64, 2 * 64) and cache_traffic(d, 1, 50) == (0, 0)
    assert MI355XARWorker(make_config(model("k_state")[0])).kv_bytes_per_block() == 0


def test_recurrence_chunks_cover_every_token_once():
    starts, lens = [3, 8, 400], [5, 300, 128]
    ch, sg = recurrence_chunks(starts, lens), recurrence_segments(starts, lens)
    assert [t for f, n, _, _ in ch for t in range(f, f + n)] == [t for s, n in zip(starts, lens) for t in range(s, s + n)]
    assert sg == [(0, 1), (1, 3), (4, 1)] and [c[2] for c in ch] == [0, 0, 1, 2, 0] and max(c[1] for c in ch) == 128


def test_heads_are_padded_where_they_lie():
    w = torch.arange(2 * 3 * 5, dtype=torch.float32).reshape(6, 5) + 1
    p = pad_head_rows(w, 2, 3, 4, 8)
    assert p.shape == (8, 8) and torch.equal(p[4:7, :5], w[3:]) and not p[3].any() and not p[:, 5:].any()
    c = pad_head_cols(w.T.contiguous(), 2, 3, 4, 6)
    assert torch.equal(c[:5], p[:, :5].T) and not c[5].any()
    assert pad_heads(torch.ones(6), 2, 3, 4).tolist() == [1, 1, 1, 0, 1, 1, 1, 0]


def test_oracle_recurrence_and_lightning():
    g = torch.Generator().manual_seed(4)
    rnd = lambda *s: torch.randn(*s, generator=g, dtype=torch.float64)  # noqa: E731
    T, H, dim, vdim, W = 6, 2, 3, 4, 5
    decay = [0.5, 0.9]
    w = dict(q=rnd(H * dim, W), k=rnd(H * dim, W), v=rnd(H * vdim, W), g=rnd(H * vdim, W), o=rnd(W, H * vdim), norm=rnd(H * vdim))
    h = rnd(T, W)
    got = D.lightning(h, w, H, dim, vdim, decay, 1e-3)
    silu = lambda z: z / (1 + math.exp(-z))  # noqa: E731
    act = lambda m, t: [silu(float(r @ h[t])) for r in m]  # noqa: E731
    for t in range(T):
        o = []
        for n in range(H):
            q = act(w["q"], t)[n * dim:(n + 1) * dim]
            for e in range(vdim):                                          # o = sum over earlier tokens of decay^(age) (q . k_j) v_j
                o.append(sum(decay[n] ** (t - j) * sum(a * b for a, b in zip(q, act(w["k"], j)[n * dim:(n + 1) * dim])) * act(w["v"], j)[n * vdim + e] for j in range(t + 1)))
        r = math.sqrt(sum(v * v for v in o) / len(o) + 1e-3)
        y = torch.tensor([v / r * float(w["norm"][i]) / (1 + math.exp(-float(w["g"][i] @ h[t]))) for i, v in enumerate(o)], dtype=torch.float64)
        assert torch.allclose(got[t], w["o"] @ y, atol=1e-9)


def test_oracle_window_attention_rotation_and_sink():
    g = torch.Generator().manual_seed(5)
    rnd = lambda *s: torch.randn(*s, generator=g, dtype=torch.float64)  # noqa: E731
    T, H, G, dim, vdim, rot, base = 7, 4, 2, 6, 3, 4, 50.0
    q, k, v, sink = rnd(T, H, dim), rnd(T, G, dim), rnd(T, G, vdim), rnd(H)
    turned = D.rotate_half(q, rot, base)
    for t in range(T):
        for n in range(H):
            for i, f in ((0, 1.0), (1, base ** -0.5)):
                z = complex(q[t, n, i], q[t, n, i + 2]) * complex(math.cos(t * f), math.sin(t * f))
                assert float(turned[t, n, i]) == pytest.approx(z.real) and float(turned[t, n, i + 2]) == pytest.approx(z.imag)
    assert torch.equal(turned[:, :, rot:], q[:, :, rot:])
    for window in (1, 3, None):
        got = D.window_attention(q, k, v, 0.4, window, sink)
        for t in range(T):
            for n in range(H):
                js = [j for j in range(t + 1) if window is None or t - j < window]
                e = [math.exp(0.4 * float(q[t, n] @ k[j, n // 2])) for j in js]
                want = sum(a * v[j, n // 2] for a, j in zip(e, js)) / (sum(e) + math.exp(float(sink[n])))
                assert torch.allclose(got[t, n], want, atol=1e-10)


def test_oracle_koronex_layer_parts():
    g = torch.Generator().manual_seed(6)
    rnd = lambda *s: torch.randn(*s, generator=g, dtype=torch.float64)  # noqa: E731
    x, y, w = rnd(2, 4), rnd(2, 4), rnd(4)
    z = 1.5 * x + y
    assert torch.allclose(D.post_norm(x, y, w, 1.5, 0.1), torch.stack([r / math.sqrt(float((r * r).mean()) + 0.1) * w for r in z]))
    s = dict(gate=rnd(3, 4), proj=rnd(4, 3), norm=rnd(4))
    e = rnd(2, 3)
    gelu = lambda u: 0.5 * u * (1 + math.tanh(math.sqrt(2 / math.pi) * (u + 0.044715 * u ** 3)))  # noqa: E731
    for t, got in enumerate(D.side_input(x, e, s, 0.1)):
        r = s["proj"] @ torch.tensor([gelu(float(s["gate"][i] @ x[t])) * float(e[t, i]) for i in range(3)], dtype=torch.float64)
        assert torch.allclose(got, r / math.sqrt(float((r * r).mean()) + 0.1) * s["norm"])
    m = dict(up=rnd(3, 4), down=rnd(4, 3))
    assert torch.allclose(D.relu2_mlp(x, m)[0], m["down"] @ torch.tensor([max(float(r @ x[0]), 0.0) ** 2 for r in m["up"]], dtype=torch.float64))
