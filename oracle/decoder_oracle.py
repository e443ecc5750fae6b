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


# ---------------------------------------------------------------- Koronex
# A decoder-only language model of two sequence mixers, norms behind the sums and a second token embedding read by every layer:
#   layer      x = norm(a x + mixer(x), w1);  x = norm(a x + ff(x), w2)  (a layer may have no feed-forward);  x += side input of the token
#   mixers     lightning: a linear recurrence with one decay per head;  attention: a sliding window, grouped key / value heads, partly rotated,
#              one extra number per head in the softmax's denominator; a layer may read an earlier layer's keys and values
#   head       logits = W norm(s, w_f), the stream starts at scale * embedding


def gelu_tanh(z: torch.Tensor) -> torch.Tensor:
    return 0.5 * z * (1 + torch.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z ** 3)))


def post_norm(x: torch.Tensor, y: torch.Tensor, w: torch.Tensor, alpha: float, eps: float) -> torch.Tensor:
    return rms_norm(alpha * x + y, w, eps)


def side_input(x: torch.Tensor, e: torch.Tensor, w: dict, eps: float) -> torch.Tensor:
    """What a token's own embedding e adds to its stream row; w: gate, proj, norm."""
    return rms_norm((gelu_tanh(x @ w["gate"].T) * e) @ w["proj"].T, w["norm"], eps)


def relu2_mlp(x: torch.Tensor, w: dict) -> torch.Tensor:
    return torch.relu(x @ w["up"].T) ** 2 @ w["down"].T


def decay_recurrence(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, decay) -> torch.Tensor:
    """q, k [T, H, D], v [T, H, E]: S <- decay S + k v^T, o = S^T q, token by token from a zero state."""
    T, H, D = q.shape
    out = torch.empty(T, H, v.shape[-1], dtype=q.dtype)
    for h in range(H):
        S = torch.zeros(D, v.shape[-1], dtype=q.dtype)
        for t in range(T):
            S = decay[h] * S + k[t, h][:, None] * v[t, h][None, :]
            out[t, h] = q[t, h] @ S
    return out


def lightning(h: torch.Tensor, w: dict, heads: int, dim: int, vdim: int, decay, eps: float) -> torch.Tensor:
    """w: q, k, v, g, o, norm."""
    T = h.shape[0]
    silu = lambda z: z * torch.sigmoid(z)  # noqa: E731
    q, k, v = silu(h @ w["q"].T).reshape(T, heads, dim), silu(h @ w["k"].T).reshape(T, heads, dim), silu(h @ w["v"].T).reshape(T, heads, vdim)
    o = decay_recurrence(q, k, v, decay).reshape(T, heads * vdim)
    return (rms_norm(o, w["norm"], eps) * torch.sigmoid(h @ w["g"].T)) @ w["o"].T


def rotate_half(x: torch.Tensor, dims: int, base: float) -> torch.Tensor:
    """x [T, H, D]: dimensions i and i + dims / 2 of the first `dims` turn by t * base^(-2 i / dims)."""
    out, half = x.clone(), dims // 2
    freq = torch.tensor([base ** (-2.0 * i / dims) for i in range(half)], dtype=torch.float64)
    for t in range(x.shape[0]):
        a = (t * freq).to(torch.float64)
        c, s = a.cos().to(x.dtype), a.sin().to(x.dtype)
        u, v = x[t, :, :half], x[t, :, half:dims]
        out[t, :, :half], out[t, :, half:dims] = u * c - v * s, v * c + u * s
    return out


def window_attention(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, scale: float, window: int | None = None, sink: torch.Tensor | None = None) -> torch.Tensor:
    """q [T, H, D], k [T, G, D], v [T, G, E] -> [T, H, E]: token i sees j <= i with i - j < window; the softmax's denominator counts exp(sink) once."""
    T, H, _ = q.shape
    G = k.shape[1]
    out = torch.empty(T, H, v.shape[-1], dtype=q.dtype)
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    seen = (j <= i) if window is None else (j <= i) & (i - j < window)
    for h in range(H):
        g = h // (H // G)
        s = (q[:, h] @ k[:, g].T * scale).masked_fill(~seen, -math.inf)
        if sink is not None:
            s = torch.cat([s, sink[h].to(s.dtype).reshape(1, 1).expand(T, 1)], 1)
        out[:, h] = torch.softmax(s, -1)[:, :T] @ v[:, g]
    return out


def attention_keys(h: torch.Tensor, w: dict, m: dict, eps: float) -> tuple[torch.Tensor, torch.Tensor]:
    """(keys behind norm and rotation, values) of a layer with projections of its own."""
    T = h.shape[0]
    k = rms_norm(h @ w["k"].T, w["k_norm"], eps).reshape(T, m["kv_heads"], m["dim"])
    return rotate_half(k, m["rot"]["dims"], m["rot"]["base"]), (h @ w["v"].T).reshape(T, m["kv_heads"], m["vdim"])


def grouped_attention(h: torch.Tensor, w: dict, m: dict, k: torch.Tensor, v: torch.Tensor, eps: float) -> torch.Tensor:
    """w: q, q_norm, sink, g, o; k, v of this layer or of the one it reads."""
    T = h.shape[0]
    q = rms_norm(h @ w["q"].T, w["q_norm"], eps).reshape(T, m["heads"], m["dim"])
    o = window_attention(rotate_half(q, m["rot"]["dims"], m["rot"]["base"]), k, v, m["scale"], m["mask"]["size"], w["sink"])
    return (o.reshape(T, -1) * torch.sigmoid(h @ w["g"].T)) @ w["o"].T


def koronex_forward(weights: dict, config: dict, tokens: list[int], dtype=torch.float32) -> tuple[torch.Tensor, list[torch.Tensor]]:
    """(logits [T, vocab], residual stream after every layer) of one whole sequence."""
    weights = {k: t.to(dtype) for k, t in weights.items()}
    eps, alpha, sd = float(config["norm"]["eps"]), float(config["postln_alpha"]), config["token_side"]["dim"]
    ids = torch.as_tensor(tokens)
    x = weights["embed"][ids] * config["embedding"]["scale"]
    trail, kv = [], {}
    for i, spec in enumerate(config["layers"]):
        own, mix, mlp = layer_tensors(weights, config, i)
        m = spec["mixer"]
        if spec["type"] == "lightning":
            y = lightning(x, mix, m["heads"], m["dim"], m["vdim"], m["decay"], eps)
        else:
            src = m.get("kv_from")
            kv[i] = kv[src] if src is not None else attention_keys(x, mix, m, eps)
            y = grouped_attention(x, mix, m, *kv[i], eps)
        x = post_norm(x, y, own["norm1"], alpha, eps)
        if spec["mlp"] is not None:
            x = post_norm(x, relu2_mlp(x, mlp), own["norm2"], alpha, eps)
        x = x + side_input(x, weights["side.embed"][ids][:, i * sd:(i + 1) * sd], {n: own["side." + n] for n in ("gate", "proj", "norm")}, eps)
        trail.append(x)
    return rms_norm(x, weights["final.norm"], eps) @ weights["head"].T, trail
