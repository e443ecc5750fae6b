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
class WindowAttentionSpec:
    """Causal attention of grouped heads over a cache of keys and values, each token seeing the last `window` tokens (itself included)."""
    heads: int
    kv_heads: int
    dim: int            # query / key dimensions per head
    vdim: int           # value dimensions per head
    scale: float        # of the scores
    window: int | None = None           # None: every earlier token
    rot_dims: int = 0                   # rotated dimensions of a head: i turns with i + rot_dims / 2
    rot_base: float = 10000.0
    qk_norm: bool = True                # RMS norms over the whole query / key projection, before the rotation
    sink: bool = False                  # one number per head in the softmax's denominator
    out_gate: bool = False              # the concatenated heads times sigmoid of a projection of the mixer's input
    kv_from: int | None = None          # the layer whose cached keys and values this one reads


@dataclass(frozen=True)
class DecayRecurrenceSpec:
    """Linear recurrence (lightning attention): S <- decay S + k v^T, o = S^T q per head, SiLU on q, k and v; all heads normed together and gated."""
    heads: int
    dim: int
    vdim: int
    decay: tuple[float, ...]            # one per head


MixerSpec = LatentAttentionSpec | WindowAttentionSpec | DecayRecurrenceSpec


@dataclass(frozen=True)
class DenseMLPSpec:
    ff: int
    act: str = "xielu"                  # or "relu2"


@dataclass(frozen=True)
class LayerSpec:
    mixer: MixerSpec
    mlp: DenseMLPSpec | None = None
    weights_of: int | None = None


@dataclass(frozen=True)
class DecoderDims:
    """Every layer: h = token shift of x (or x); the mixer's and the feed-forward's outputs join the stream through `norm`:
      "output"   x += g y / rms(y), one number g per norm;   the head reads g_f x / rms(x)
      "post"     x = w z / rms(z), z = alpha x + y, a weight vector w per norm;   likewise the head
    side_dim > 0: every layer ends with x += w_s r / rms(r), r = W_p (gelu(W_g x) * e), e the layer's slice of a second embedding of the token."""
    name: str
    hidden: int
    vocab: int
    layers: tuple[LayerSpec, ...]
    eps: float
    max_model_len: int = 4096
    norm: str = "output"
    alpha: float = 1.0
    token_shift: bool = True
    embed_scale: float = 1.0
    side_dim: int = 0

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

    def kv_owner(self, i: int) -> int | None:
        """The layer whose cached keys and values layer i's mixer reads (None: it keeps none)."""
        m = self.layers[i].mixer
        if isinstance(m, DecayRecurrenceSpec):
            return None
        return i if getattr(m, "kv_from", None) is None else m.kv_from

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


def _object(d: dict, what: str, key: str) -> dict:
    if not isinstance(d.get(key), dict):
        raise ValueError(f"{what}: missing object {key!r}")
    return d[key]


def _koronex_mixer(e: dict, i: int, what: str) -> MixerSpec:
    m = _object(e, what, "mixer")
    what += ".mixer"
    if e["type"] == "lightning":
        m = _take(m, what, dict(heads=int, dim=int, vdim=int, decay=lambda v: tuple(float(f) for f in v)))
        _positive(**{k: m[k] for k in ("heads", "dim", "vdim")})
        if len(m["decay"]) != m["heads"] or min(m["decay"]) <= 0:
            raise ValueError(f"{what}: one positive decay per head")
        return DecayRecurrenceSpec(**m)
    m = _take(m, what, dict(heads=int, kv_heads=int, dim=int, vdim=int, scale=float, mask=dict, rot=dict), dict(kv_from=lambda v: None if v is None else int(v)))
    mask, rot = _take(m.pop("mask"), what + ".mask", dict(size=int)), _take(m.pop("rot"), what + ".rot", dict(base=float, dims=int))
    _positive(**{k: m[k] for k in ("heads", "kv_heads", "dim", "vdim")}, **mask, base=rot["base"])
    if m["heads"] % m["kv_heads"]:
        raise ValueError(f"{what}: {m['heads']} heads over {m['kv_heads']} key / value heads")
    if not 0 <= rot["dims"] <= m["dim"] or rot["dims"] % 2:
        raise ValueError(f"{what}: {rot['dims']} rotated dimensions of {m['dim']}")
    if m.get("kv_from") is not None and not 0 <= m["kv_from"] < i:
        raise ValueError(f"{what}: kv_from {m['kv_from']} is not an earlier layer")
    return WindowAttentionSpec(**m, window=mask["size"], rot_dims=rot["dims"], rot_base=rot["base"], sink=True, out_gate=True)


def parse_koronex(cfg: dict, max_model_len: int = 4096) -> DecoderDims:
    layers = []
    for i, e in enumerate(cfg["layers"]):
        what = f"layers[{i}]"
        if e.get("type") not in ("lightning", "attention"):
            raise ValueError(f"{what}: mixer type {e.get('type')!r} (known: 'attention', 'lightning')")
        extra = set(e) - {"type", "mixer", "mlp"}
        if extra:
            raise ValueError(f"{what}: unknown {sorted(extra)}")
        mlp = e.get("mlp")
        if mlp is not None:
            mk = _take(mlp, f"{what}.mlp", dict(kind=str, ff=int))
            if mk["kind"] != "dense":
                raise ValueError(f"{what}.mlp: kind {mk['kind']!r} (known: 'dense')")
            _positive(ff=mk["ff"])
            mlp = DenseMLPSpec(ff=mk["ff"], act="relu2")
        layers.append(LayerSpec(_koronex_mixer(e, i, what), mlp))
    d = DecoderDims(name="koronex", hidden=int(cfg["width"]), vocab=int(cfg["vocab"]), layers=tuple(layers), eps=float(cfg["norm"]["eps"]),
                    max_model_len=int(max_model_len), norm="post", alpha=float(cfg["postln_alpha"]), token_shift=False,
                    embed_scale=float(cfg["embedding"]["scale"]), side_dim=int(cfg["token_side"]["dim"]))
    _positive(width=d.hidden, vocab=d.vocab, layers=d.num_layers, side_dim=d.side_dim)
    for i, s in enumerate(d.layers):
        src = getattr(s.mixer, "kv_from", None)
        if src is None:
            continue
        o = d.layers[src].mixer
        same = ("kv_heads", "dim", "vdim", "rot_dims", "rot_base")
        if not isinstance(o, WindowAttentionSpec) or o.kv_from is not None or any(getattr(o, k) != getattr(s.mixer, k) for k in same):
            raise ValueError(f"layers[{i}] reads the keys and values of layers[{src}], which has none of its own or of another shape")
    return d


PARSERS = {"Zefedra": parse_zefedra, "Koronex": parse_koronex}


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


def _mixer_shapes(m: MixerSpec, W: int) -> dict[str, tuple[int, ...]]:
    """Tensors of a mixer, names without the layer's prefix."""
    if isinstance(m, LatentAttentionSpec):
        out = {"dq": (m.q_rank, W), "dq.norm": (m.q_rank,), "uq": (m.heads * m.dim, m.q_rank), "dkv": (m.kv_rank, W), "dkv.norm": (m.kv_rank,),
               "uk": (m.heads * m.dim, m.kv_rank), "uv": (m.heads * m.vdim, m.kv_rank), "o": (W, m.heads * m.vdim)}
        return {**out, "g": (m.heads, W)} if m.out_gate else out
    if isinstance(m, DecayRecurrenceSpec):
        n = m.heads * m.vdim
        return {"q": (m.heads * m.dim, W), "k": (m.heads * m.dim, W), "v": (n, W), "g": (n, W), "o": (W, n), "norm": (n,)}
    q, k, v = m.heads * m.dim, m.kv_heads * m.dim, m.heads * m.vdim
    out = {"q": (q, W), "o": (W, v)}
    if m.kv_from is None:
        out.update({"k": (k, W), "v": (m.kv_heads * m.vdim, W)})
    if m.qk_norm:
        out["q.norm"] = (q,)
        if m.kv_from is None:
            out["k.norm"] = (k,)
    if m.sink:
        out["sink"] = (m.heads,)
    if m.out_gate:
        out["g"] = (v, W)
    return out


def tensor_shapes(d: DecoderDims) -> dict[str, tuple[int, ...]]:
    """Checkpoint tensor names and shapes of a model (layers that borrow have none)."""
    W = d.hidden
    norm = (W,) if d.norm == "post" else ()
    out: dict[str, tuple[int, ...]] = {"embed": (d.vocab, W), "final.norm": norm, "head": (d.vocab, W)}
    if d.side_dim:
        out["side.embed"] = (d.vocab, d.num_layers * d.side_dim)
    for i, s in enumerate(d.layers):
        if s.weights_of is not None:
            continue
        p = f"l{i}."
        out[p + "norm1"] = norm
        if d.token_shift:
            out[p + "shift"] = (W,)
        out.update({p + "mix." + k: shape for k, shape in _mixer_shapes(s.mixer, W).items()})
        if s.mlp is not None:
            out.update({p + "norm2": norm, p + "mlp.up": (s.mlp.ff, W), p + "mlp.down": (W, s.mlp.ff)})
            if s.mlp.act == "xielu":
                out[p + "mlp.act"] = (2,)
        if d.side_dim:
            out.update({p + "side.gate": (d.side_dim, W), p + "side.proj": (W, d.side_dim), p + "side.norm": (W,)})
    return out
