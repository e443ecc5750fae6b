"""Small Zefedra and Koronex models of the tests' own: configurations, random weights in checkpoint naming, and what the oracle says about them."""
from __future__ import annotations

import torch

from ht_vllm_omni_amd.decoder_config import dims_from_config
from ht_vllm_omni_amd.weights import make_decoder_weights
from oracle import decoder_oracle as D


def layer(kind="latent_attention", heads=3, dim=24, vdim=40, kv_rank=56, q_rank=48, scale=0.21, ff=104, weights_of=None):
    e = {"type": kind, "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "kv_rank": kv_rank, "q_rank": q_rank, "scale": scale},
         "mlp": None if ff is None else {"kind": "dense", "ff": ff}}
    if weights_of is not None:
        e["weights_of"] = weights_of
    return e


def config(layers, width=136, vocab=203, eps=1e-5):
    return {"architecture": "Zefedra", "width": width, "vocab": vocab, "norm": {"eps": eps}, "layers": layers}


G = "latent_attention_2"
CONFIGS = {
    # odd sizes, both mixers, a layer without feed-forward, borrowed layers whose owner comes before and after
    "mixed": config([layer(), layer(G, heads=5, dim=16, vdim=8, kv_rank=72, q_rank=40, scale=0.3, ff=None), layer(weights_of=0),
                     layer(G, heads=5, dim=16, vdim=8, kv_rank=72, q_rank=40, scale=0.3, ff=None, weights_of=1)]),
    # one head, width-one ranks' neighbours, heads = dim = vdim
    "narrow": config([layer(G, heads=1, dim=8, vdim=8, kv_rank=8, q_rank=8, scale=0.3, ff=24), layer(heads=8, dim=8, vdim=8, kv_rank=32, q_rank=16, scale=0.25, ff=32)],
                     width=40, vocab=50, eps=1e-6),
    # more heads than one 16-row tile, wide latents
    "wide": config([layer(heads=20, dim=32, vdim=24, kv_rank=264, q_rank=160, scale=0.18, ff=320), layer(G, heads=16, dim=96, vdim=64, kv_rank=512, q_rank=96, scale=0.1, ff=224)],
                   width=320, vocab=331),
    # gated layers only, the owner of a borrowed layer sits behind it
    "behind": config([layer(G, heads=2, ff=64, weights_of=1), layer(G, heads=2, ff=64)], width=96, vocab=77),
}


def lightning(heads=3, dim=24, vdim=40, decay=None, ff=None):
    decay = [0.5 + 0.4995 * h / max(heads - 1, 1) for h in range(heads)] if decay is None else decay
    return {"type": "lightning", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": decay}, "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def attention(heads=6, kv_heads=2, dim=40, vdim=24, scale=0.17, window=9, rot=16, base=1e4, kv_from=None, ff=88):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "mask": {"size": window}, "rot": {"base": base, "dims": rot}}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "attention", "mixer": m, "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def koronex(layers, width=104, vocab=211, eps=1e-5, alpha=1.7, scale=2.0, side=10):
    return {"architecture": "Koronex", "width": width, "vocab": vocab, "norm": {"eps": eps}, "postln_alpha": alpha, "embedding": {"scale": scale},
            "token_side": {"dim": side}, "layers": layers}


KORONEX = {
    # both mixers with and without feed-forward, shared keys under other windows and scales, as many key / value heads as heads, every dimension rotated
    "k_mixed": koronex([attention(ff=None), lightning(ff=72), attention(kv_from=0, window=20, scale=0.3), lightning(heads=2, dim=40, vdim=16), attention(4, 4, 16, 16, 0.25, 70, 16, 500.0),
                        attention(4, 4, 16, 16, 0.25, 3, 16, 500.0, kv_from=4, ff=None)], alpha=2.4, side=40),
    # one of everything, a window of one token, norms of a sum that weighs the stream less
    "k_narrow": koronex([attention(1, 1, 8, 8, 0.5, 1, 2, 10.0, ff=8), lightning(1, 8, 8, [0.75], ff=24), attention(1, 1, 8, 8, 0.5, 30, 6, 100.0, ff=16)],
                        width=40, vocab=50, eps=1e-6, alpha=2.0, scale=1.0, side=28),
    # more grouped heads than one 16-row tile, heads wider than 128, values wider than one column block
    "k_wide": koronex([lightning(2, 136, 200, [0.9, 0.997], ff=160), attention(20, 1, 72, 136, 0.1, 33, 36, ff=224), attention(24, 3, 128, 128, 0.09, 150, 64, ff=None)],
                      width=320, vocab=331, alpha=2.2, side=72),
    # heads wider than the matrix-core kernels take
    "k_plain": koronex([attention(2, 1, 264, 288, 0.06, 17, 20, ff=40), lightning(1, 264, 288, [0.98])], width=72, vocab=90, alpha=1.0, side=32),
    # nothing is cached
    "k_state": koronex([lightning(2, 16, 8, [1.0, 0.125], ff=32), lightning(4, 8, 32)], width=64, vocab=65, side=30),
}
CONFIGS.update(KORONEX)


def model(name, seed=0, sharp=1.0, max_model_len=2048):
    """(dims, weights, config); sharp > 1 scales the keys so that single keys decide the softmax."""
    cfg = CONFIGS[name]
    d = dims_from_config(cfg, max_model_len)
    w = make_decoder_weights(d, seed=seed)
    if sharp != 1.0:
        for k in w:
            if k.endswith(("mix.uk", "mix.k.norm")):
                w[k] = (w[k].float() * sharp).to(torch.bfloat16)
    # (a side input is normed, too: widths of a few dimensions would do the same to it)
    # a recurrence's output is normed whatever its size: queries that resemble the keys keep it away from zero, where its direction is rounding
    for i, e in enumerate(cfg["layers"]):
        if e["type"] == "lightning":
            q, k = w[f"l{i}.mix.q"].float(), w[f"l{i}.mix.k"].float()
            w[f"l{i}.mix.q"] = (0.6 * q + 0.8 * k).to(torch.bfloat16)
    return d, w, cfg


def tokens(n, vocab, seed=0):
    return torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(1000 + seed)).tolist()


def oracle(w, cfg, toks, dtype=torch.float32):
    """(logits, residual stream behind every layer)"""
    return {"Zefedra": D.zefedra_forward, "Koronex": D.koronex_forward}[cfg["architecture"]](w, cfg, toks, dtype)


def oracle_logits(w, cfg, toks, dtype=torch.float32):
    return oracle(w, cfg, toks, dtype)[0]


TOL = {"float32": 2e-5, "bfloat16": 4e-2}


def assert_logits(got, ref, dtype, what=""):
    """Every row's rms difference against the rms of all logits."""
    g, r = got.float().cpu(), ref.float()
    assert g.shape == r.shape, (what, g.shape, r.shape)
    err = (g - r).pow(2).mean(-1).sqrt() / r.pow(2).mean().sqrt()
    assert torch.isfinite(g).all() and float(err.max()) <= TOL[dtype], f"{what}: row {int(err.argmax())} of {len(err)} is off by {float(err.max()):.3g} (limit {TOL[dtype]})"
