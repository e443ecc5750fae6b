"""Dimensions of decoder-only language models described layer by layer (config.json key ``layers``).

A model is a list of ``LayerSpec``: a sequence mixer, an optional feed-forward, and whether the layer borrows another layer's tensors
(``weights_of``: same weights, its own place in the cache and the state).  Mixers and feed-forwards are small specs of their own, so a
design is a choice of specs plus the constants of its norms; ``PARSERS`` maps config.json's ``architecture`` to the function that makes it.
"""
from __future__ import annotations

import json
import os
from dataclasses import dataclass, replace


@dataclass(frozen=True)
class LatentAttentionSpec:
    """Causal attention over a cache of latents: keys and values of every head are linear in one shared vector per token; no positions."""
    heads: int
    dim: int            # query / key dimensions per head
    vdim: int           # value dimensions per head
    q_rank: int         # width of the query latent
    kv_rank: int        # width of the cached latent
    scale: float        # of the scores
    out_gate: bool = False      # each head's output times sigmoid of a projection of the mixer's input


@dataclass(frozen=True)
class DenseMLPSpec:
    ff: int
    act: str = "xielu"


@dataclass(frozen=True)
class LayerSpec:
    mixer: LatentAttentionSpec
    mlp: DenseMLPSpec | None = None
    weights_of: int | None = None


@dataclass(frozen=True)
class DecoderDims:
    """Every layer: h = token shift of x; x += norm(mixer(h)); x += norm(mlp(x)); norms are RMS with one gain each (on the outputs only)."""
    name: str
    hidden: int
    vocab: int
    layers: tuple[LayerSpec, ...]
    eps: float
    max_model_len: int = 4096

    @property
    def num_layers(self) -> int:
        return len(self.layers)

    def owner(self, i: int) -> int:
        """The layer whose tensors layer i uses (itself, or the end of its ``weights_of`` chain)."""
        seen = set()
        while self.layers[i].weights_of is not None:
            if i in seen:
                raise ValueError(f"layers {sorted(seen)} borrow each other's weights in a circle")
            seen.add(i)
            i = self.layers[i].weights_of
        return i

    def with_(self, **kw) -> "DecoderDims":
        return replace(self, **kw)


def _take(d: dict, what: str, required: dict, optional: dict | None = None) -> dict:
    """The named keys of a config object, converted; a key that is missing or that nothing here reads is an error, not a guess."""
    optional = optional or {}
    extra = set(d) - set(required) - set(optional)
    missing = set(required) - set(d)
    if extra or missing:
        raise ValueError(f"{what}: " + "; ".join(filter(None, (f"missing {sorted(missing)}" if missing else "", f"unknown {sorted(extra)}" if extra else ""))))
    return {k: conv(d[k]) for k, conv in {**required, **{k: c for k, c in optional.items() if k in d}}.items()}


def _positive(**kw) -> None:
    for k, v in kw.items():
        if v <= 0:
            raise ValueError(f"{k} = {v} must be positive")


# Zefedra's two mixer types: latent attention, without and with the per-head output gate
_ZEFEDRA_MIXERS = {"latent_attention": False, "latent_attention_2": True}


def parse_zefedra(cfg: dict, max_model_len: int = 4096) -> DecoderDims:
    layers = []
    n = len(cfg["layers"])
    for i, e in enumerate(cfg["layers"]):
        what = f"layers[{i}]"
        if e.get("type") not in _ZEFEDRA_MIXERS:
            raise ValueError(f"{what}: mixer type {e.get('type')!r} (known: {sorted(_ZEFEDRA_MIXERS)})")
        m = _take(e["mixer"], f"{what}.mixer", dict(heads=int, dim=int, vdim=int, kv_rank=int, q_rank=int, scale=float))
        _positive(**{k: m[k] for k in ("heads", "dim", "vdim", "kv_rank", "q_rank")})
        mlp = e.get("mlp")
        if mlp is not None:
            mk = _take(mlp, f"{what}.mlp", dict(kind=str, ff=int))
            if mk["kind"] != "dense":
                raise ValueError(f"{what}.mlp: kind {mk['kind']!r} (known: 'dense')")
            _positive(ff=mk["ff"])
            mlp = DenseMLPSpec(ff=mk["ff"])
        src = e.get("weights_of")
        if src is not None and not 0 <= int(src) < n:
            raise ValueError(f"{what}: weights_of {src} is not a layer")
        layers.append(LayerSpec(LatentAttentionSpec(out_gate=_ZEFEDRA_MIXERS[e["type"]], **m), mlp, None if src is None else int(src)))
    d = DecoderDims(name="zefedra", hidden=int(cfg["width"]), vocab=int(cfg["vocab"]), layers=tuple(layers), eps=float(cfg["norm"]["eps"]),
                    max_model_len=int(max_model_len))
    _positive(width=d.hidden, vocab=d.vocab, layers=n)
    for i, s in enumerate(d.layers):
        o = d.layers[d.owner(i)]
        if (s.mixer, s.mlp) != (o.mixer, o.mlp):
            raise ValueError(f"layers[{i}] borrows the weights of layers[{d.owner(i)}] but differs from it")
    return d


PARSERS = {"Zefedra": parse_zefedra}


def read_config(path: str | dict) -> dict:
    """config.json as a dict, from a dict, a file or a model directory."""
    if isinstance(path, dict):
        return path
    if os.path.isdir(path):
        path = os.path.join(path, "config.json")
    with open(path) as f:
        return json.load(f)


def dims_from_config(cfg: str | dict, max_model_len: int = 4096) -> DecoderDims:
    cfg = read_config(cfg)
    arch = cfg.get("architecture")
    if arch not in PARSERS:
        raise ValueError(f"architecture {arch!r} is not a decoder-only model of this package (known: {sorted(PARSERS)})")
    return PARSERS[arch](cfg, max_model_len)


def tensor_shapes(d: DecoderDims) -> dict[str, tuple[int, ...]]:
    """Checkpoint tensor names and shapes of a model (layers that borrow have none)."""
    W = d.hidden
    out: dict[str, tuple[int, ...]] = {"embed": (d.vocab, W), "final.norm": (), "head": (d.vocab, W)}
    for i, s in enumerate(d.layers):
        if s.weights_of is not None:
            continue
        p, m = f"l{i}.", s.mixer
        out.update({p + "norm1": (), p + "shift": (W,),
                    p + "mix.dq": (m.q_rank, W), p + "mix.dq.norm": (m.q_rank,), p + "mix.uq": (m.heads * m.dim, m.q_rank),
                    p + "mix.dkv": (m.kv_rank, W), p + "mix.dkv.norm": (m.kv_rank,), p + "mix.uk": (m.heads * m.dim, m.kv_rank),
                    p + "mix.uv": (m.heads * m.vdim, m.kv_rank), p + "mix.o": (W, m.heads * m.vdim)})
        if m.out_gate:
            out[p + "mix.g"] = (m.heads, W)
        if s.mlp is not None:
            out.update({p + "norm2": (), p + "mlp.up": (s.mlp.ff, W), p + "mlp.down": (W, s.mlp.ff), p + "mlp.act": (2,)})
    return out
