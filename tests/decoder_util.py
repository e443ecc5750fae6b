"""Small Zefedra models of the tests' own: configurations, random weights in checkpoint naming, and what the oracle says about them."""
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


def model(name, seed=0, sharp=1.0, max_model_len=2048):
    """(dims, weights, config); sharp > 1 scales the keys' product so that single keys decide the softmax."""
    cfg = CONFIGS[name]
    d = dims_from_config(cfg, max_model_len)
    w = make_decoder_weights(d, seed=seed)
    if sharp != 1.0:
        for k in w:
            if k.endswith("mix.uk"):
                w[k] = (w[k].float() * sharp).to(torch.bfloat16)
    return d, w, cfg


def tokens(n, vocab, seed=0):
    return torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(1000 + seed)).tolist()


def oracle_logits(w, cfg, toks, dtype=torch.float32):
    return D.zefedra_forward(w, cfg, toks, dtype)[0]


TOL = {"float32": 2e-5, "bfloat16": 4e-2}


def assert_logits(got, ref, dtype, what=""):
    """Every row's rms difference against the rms of all logits."""
    g, r = got.float().cpu(), ref.float()
    assert g.shape == r.shape, (what, g.shape, r.shape)
    err = (g - r).pow(2).mean(-1).sqrt() / r.pow(2).mean().sqrt()
    assert torch.isfinite(g).all() and float(err.max()) <= TOL[dtype], f"{what}: row {int(err.argmax())} of {len(err)} is off by {float(err.max()):.3g} (limit {TOL[dtype]})"
