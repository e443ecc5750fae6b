"""Plain restatement of the decoder-only designs the language-model engine serves (test oracle: slow, no cache, no batch).

One function per mechanism, written from its equations on whole sequences in the dtype of the inputs (the tests use fp32 and fp64);
nothing here imports the package.  Rows of `x` are the tokens of ONE sequence in order; linear weights are [out, in].

Zefedra -- a decoder-only language model without position encodings:
  layer      h = shift(x);  x += norm(mixer(h), g1);  x += norm(ff(x), g2)          (a layer may have no feed-forward)
  norm       y / sqrt(mean(y^2) + eps) * g with ONE number g                          (scalar_rms_norm)
  shift      h_t = x_t + (x_{t-1} - x_t) * mu, x_{-1} = 0                             (token_shift)
  mixer      queries and keys / values from latents, each RMS-normed with a plain weight vector; k, v per head from the shared
             latent c; causal softmax; optionally each head times sigmoid of a projection of h          (latent_attention)
  ff         W_down xielu(W_up x)                                                     (xielu_mlp)
  head       logits = W norm(x, g_f)
A layer may borrow another layer's tensors (same function, its own place in the sequence of layers).
"""
from __future__ import annotations

import math

import torch


def rms_norm(x: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


def scalar_rms_norm(x: torch.Tensor, g: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * g.reshape(())


def token_shift(x: torch.Tensor, mu: torch.Tensor) -> torch.Tensor:
    prev = torch.zeros_like(x)
    prev[1:] = x[:-1]
    return x + (prev - x) * mu


def causal_softmax_attention(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, scale: float) -> torch.Tensor:
    """q, k [T, H, D], v [T, H, E] -> [T, H, E]."""
    T, H, _ = q.shape
    out = torch.empty(T, H, v.shape[-1], dtype=q.dtype)
    future = torch.ones(T, T, dtype=torch.bool).triu(1)
    for h in range(H):
        s = q[:, h] @ k[:, h].T * scale
        s = s.masked_fill(future, -math.inf)
        out[:, h] = torch.softmax(s, -1) @ v[:, h]
    return out


def latent_attention(h: torch.Tensor, w: dict, heads: int, dim: int, vdim: int, scale: float, eps: float, gated: bool) -> torch.Tensor:
    """w: dq, dq_norm, uq, dkv, dkv_norm, uk, uv, o and, when gated, g."""
    T = h.shape[0]
    q = (rms_norm(h @ w["dq"].T, w["dq_norm"], eps) @ w["uq"].T).reshape(T, heads, dim)
    c = rms_norm(h @ w["dkv"].T, w["dkv_norm"], eps)
    k = (c @ w["uk"].T).reshape(T, heads, dim)
    v = (c @ w["uv"].T).reshape(T, heads, vdim)
    o = causal_softmax_attention(q, k, v, scale)
    if gated:
        o = o * torch.sigmoid(h @ w["g"].T)[:, :, None]
    return o.reshape(T, heads * vdim) @ w["o"].T


def xielu(z: torch.Tensor, pq: torch.Tensor) -> torch.Tensor:
    a, b = (torch.log1p(torch.exp(-v.abs())) + v.clamp_min(0) for v in pq.to(z.dtype))      # softplus
    return torch.where(z > 0, a * z * z + z / 2, (0.5 + b) * (torch.expm1(z.clamp_max(0)) - z) + z / 2)


def xielu_mlp(x: torch.Tensor, w: dict) -> torch.Tensor:
    return xielu(x @ w["up"].T, w["act"]) @ w["down"].T


def layer_tensors(weights: dict, config: dict, i: int) -> tuple[dict, dict, dict]:
    """(own tensors of layer i or of the layer it borrows from, its mixer's, its feed-forward's), names without the prefix."""
    while config["layers"][i].get("weights_of") is not None:
        i = config["layers"][i]["weights_of"]
    p = f"l{i}."
    own = {k[len(p):]: t for k, t in weights.items() if k.startswith(p)}
    mix = {k[4:].replace(".norm", "_norm"): t for k, t in own.items() if k.startswith("mix.")}
    mlp = {k[4:]: t for k, t in own.items() if k.startswith("mlp.")}
    return own, mix, mlp


def zefedra_forward(weights: dict, config: dict, tokens: list[int], dtype=torch.float32) -> tuple[torch.Tensor, list[torch.Tensor]]:
    """(logits [T, vocab], residual stream after every layer) of one whole sequence."""
    weights = {k: t.to(dtype) for k, t in weights.items()}
    eps = float(config["norm"]["eps"])
    x = weights["embed"][torch.as_tensor(tokens)]
    trail = []
    for i, spec in enumerate(config["layers"]):
        own, mix, mlp = layer_tensors(weights, config, i)
        m = spec["mixer"]
        h = token_shift(x, own["shift"])
        gated = {"latent_attention": False, "latent_attention_2": True}[spec["type"]]
        y = latent_attention(h, mix, m["heads"], m["dim"], m["vdim"], m["scale"], eps, gated)
        x = x + scalar_rms_norm(y, own["norm1"], eps)
        if spec["mlp"] is not None:
            x = x + scalar_rms_norm(xielu_mlp(x, mlp), own["norm2"], eps)
        trail.append(x)
    return scalar_rms_norm(x, weights["final.norm"], eps) @ weights["head"].T, trail
