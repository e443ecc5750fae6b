"""Sequence mixers of the decoder-only language models: weights on the device, cache and state of a layer, launches.

A mixer object belongs to the layer that owns the weights; ``run(engine, b, i, s, x, frag)`` runs it as layer ``i`` (a borrowing layer has its own place in the
cache and the state) on the operand ``s.h`` and returns how many partial sums its output ``s.y`` consists of.  ``needs`` names the
activations it wants per token; every layer of a model shares them (``decoder_engine._Scratch``).  ``work`` names the lists of work items its
kernels walk, one builder per kind (``WORK``), made once per batch.

  LatentMixer   latent attention over a paged cache of latents (csrc/latent_attn.hip)
  WindowMixer   grouped, rotated attention with an optional window, sink and gate over paged keys and values, its own or an earlier layer's
                (csrc/window_attn.hip)
  DecayMixer    linear recurrence with one decay per head and an fp32 state per sequence (csrc/decay_rec.hip)
"""
from __future__ import annotations

import ctypes as C
import math
from dataclasses import dataclass

import torch

from . import _lib as L
from .decoder_config import DecayRecurrenceSpec, DecoderDims, LatentAttentionSpec, WindowAttentionSpec
from .engine import frag_shuffle


@dataclass(frozen=True)
class Elem:
    code: int
    torch: torch.dtype
    kv_names: tuple[str, ...]


ELEM = {"bfloat16": Elem(0, torch.bfloat16, ("auto", "bf16", "bfloat16")), "float32": Elem(1, torch.float32, ("auto", "float32", "fp32"))}


def r32(n: int) -> int:
    return (n + 31) // 32 * 32


# latent widths the matrix-core attention is instantiated for (csrc/latent_attn.hip LA_WIDTHS)
LATENT_WIDTHS = tuple(32 * n for n in (1, 2, 3, 4, 5, 6, 7, 8, 10, 12, 14, 16))


def latent_width(kv_rank: int, elem_code: int) -> int:
    """Padded width of a cache row."""
    if elem_code == 0:
        for w in LATENT_WIDTHS:
            if w >= kv_rank:
                return w
    return r32(kv_rank)


def pad2(w: torch.Tensor, rows: int, cols: int) -> torch.Tensor:
    out = torch.zeros(rows, cols, dtype=w.dtype, device=w.device)
    out[:w.shape[0], :w.shape[1]] = w
    return out


def pad1(v: torch.Tensor, n: int) -> torch.Tensor:
    out = torch.zeros(n, dtype=v.dtype, device=v.device)
    out[:v.shape[0]] = v
    return out


def pad_head_rows(w: torch.Tensor, heads: int, dim: int, dp: int, cols: int) -> torch.Tensor:
    """[heads * dim, K] -> [heads * dp, cols], every head's rows padded."""
    return torch.cat([pad2(h, dp, cols) for h in w.reshape(heads, dim, w.shape[1])])


def pad_head_cols(w: torch.Tensor, heads: int, dim: int, dp: int, rows: int) -> torch.Tensor:
    """[N, heads * dim] -> [rows, heads * dp], every head's columns padded."""
    return torch.cat([pad2(w[:, h * dim:(h + 1) * dim], rows, dp) for h in range(heads)], 1)


def pad_heads(v: torch.Tensor, heads: int, dim: int, dp: int) -> torch.Tensor:
    """[heads * dim] -> [heads * dp]."""
    return torch.cat([pad1(h, dp) for h in v.reshape(heads, dim)])


class Matrix:
    """One weight [N, K] (or [heads, N, K]) of a layer, padded, on the device: fragment-major in bf16, row-major in fp32."""

    def __init__(self, w: torch.Tensor, elem: Elem, device):
        w = w.to(device=device, dtype=elem.torch).contiguous()
        self.t = frag_shuffle(w) if elem.code == 0 else w
        self.N, self.K = w.shape[-2:]


# ---------------------------------------------------------------- work items of a batch's segments of more than one token
def attention_tiles(seg_starts: list[int], seg_lens: list[int], heads: int, tile_rows: int) -> list[tuple[int, int]]:
    """Work items of the prompt attention: runs of up to `tile_rows` query rows (token-major, heads inside) of ONE sequence.  Longest first: a later
    tile of a prompt sees more keys."""
    out = []
    for s, n in zip(seg_starts, seg_lens):
        lo, hi = s * heads, (s + n) * heads
        out += [(lo - f, f, min(tile_rows, hi - f)) for f in range(lo, hi, tile_rows)]
    return [(f, n) for _, f, n in sorted(out)]


def recurrence_chunks(seg_starts: list[int], seg_lens: list[int]) -> list[tuple[int, int, int, int]]:
    """(first token, count, index in the segment, 0) of every chunk, segment after segment."""
    return [(s + o, min(L.REC_CHUNK, n - o), o // L.REC_CHUNK, 0) for s, n in zip(seg_starts, seg_lens) for o in range(0, n, L.REC_CHUNK)]


def recurrence_segments(seg_starts: list[int], seg_lens: list[int]) -> list[tuple[int, int]]:
    """(first chunk, chunks) of every segment."""
    out, at = [], 0
    for n in seg_lens:
        k = -(-n // L.REC_CHUNK)
        out.append((at, k))
        at += k
    return out


def recurrence_runs(seg_starts: list[int], seg_lens: list[int]) -> list[tuple[int, int]]:
    return list(zip(seg_starts, seg_lens))


# kind -> builder of its items from (segment starts, segment lengths, *parameters); a work key is (kind, *parameters)
WORK = {"tiles": attention_tiles, "chunks": recurrence_chunks, "segs": recurrence_segments, "runs": recurrence_runs}


class Mixer:
    """What the engine asks of a mixer; `eng` / `e` is the DecoderEngine (products, cache, state, block table) -- handed in, never kept: an engine that
    goes out of use gives its memory back at once."""
    work: tuple = ()

    def __init__(self, spec):
        self.spec = spec

    def cache(self, eng, num_blocks: int, block_size: int) -> tuple[torch.Tensor, ...]:
        """Cache tensors of one layer (none: nothing is paged)."""
        return ()

    def state(self, eng, slots: int) -> torch.Tensor | None:
        """State of one layer, one entry per slot."""
        return None

    def workspace_bytes(self, eng, rows: int) -> int:
        """Of the decode attention's KV splits."""
        return 0

    def needs(self) -> dict[str, tuple]:
        """Activations: name -> (elements per token, dtype or "elem", "rows" | "tiles" of 16 rows | "slabs" of partial sums)."""
        return {}

    @staticmethod
    def _where(e, b) -> dict:
        return dict(block_table=e.block_table.data_ptr(), bt_stride=e.bt_stride, block_size=e.block_size, row_of_tok=b.row_of_tok.data_ptr(),
                    positions=b.positions.data_ptr())

    @staticmethod
    def _launch(e, name: str, s) -> None:
        L.check(getattr(e.lib, name + "_run")(C.byref(s), L.current_stream()), name, e.lib)


class LatentMixer(Mixer):
    def __init__(self, eng, i: int, m: LatentAttentionSpec, w: dict):
        super().__init__(m)
        elem, dev, W, H = eng.elem, eng.device, eng.width, m.heads
        self.qp, self.rp, self.dp, self.vp = r32(m.q_rank), latent_width(m.kv_rank, elem.code), r32(m.dim), r32(m.vdim)
        parts = [pad2(w["dq"], self.qp, W), pad2(w["dkv"], self.rp, W)]
        if m.out_gate:
            parts.append(pad2(w["g"], r32(H), W))
        self.down = Matrix(torch.cat(parts), elem, dev)
        self.qw, self.kw = eng.up(pad1(w["dq.norm"], self.qp)), eng.up(pad1(w["dkv.norm"], self.rp))
        self.uq = Matrix(pad_head_rows(w["uq"], H, m.dim, self.dp, self.qp), elem, dev)
        # per head: queries into the latent space (the transpose of W_uk) and latents to values
        self.uk = Matrix(torch.stack([pad2(h.T, self.rp, self.dp) for h in w["uk"].reshape(H, m.dim, m.kv_rank)]), elem, dev)
        self.uv = Matrix(torch.stack([pad2(h, self.vp, self.rp) for h in w["uv"].reshape(H, m.vdim, m.kv_rank)]), elem, dev)
        self.o = Matrix(pad_head_cols(w["o"], H, m.vdim, self.vp, W), elem, dev)
        self.tiles = ("tiles", H, eng.lib.omni_latent_attn_tile_rows(self.rp))
        self.work = (self.tiles,)

    def matrices(self):
        return [self.down, self.uq, self.uk, self.uv, self.o]

    def cache(self, eng, num_blocks, block_size):
        return (torch.zeros(num_blocks, block_size, self.rp, dtype=eng.elem.torch, device=eng.device),)

    def workspace_bytes(self, eng, rows):
        return eng.lib.omni_latent_attn_workspace_bytes(rows, self.spec.heads, self.rp)

    def needs(self):
        H = self.spec.heads
        return {"proj": (self.down.N, torch.float32, "slabs"), "cq": (self.qp, "elem", "tiles"), "q": (H * self.dp, "elem", "rows"), "ql": (H * self.rp, "elem", "rows"),
                "ol": (H * self.rp, "elem", "rows"), "v": (H * self.vp, "elem", "tiles"), "head_gate": (H, torch.float32, "rows")}

    def run(self, e, b, i, s, x, frag):
        m = self.spec
        T, H, (cache,) = b.T, m.heads, e.kv_caches[i]
        slabs = e._mm(s.h, self.down, s.proj, T, f32_out=True)
        gate = s.head_gate if m.out_gate else None
        shift = e.shift_state
        self._launch(e, "omni_latent_write", L.LatentWrite(
            proj=s.proj.data_ptr(), slabs=slabs, slab_stride=T * self.down.N, ld=self.down.N, q_rank=m.q_rank, qp=self.qp, kv_rank=m.kv_rank, rp=self.rp, heads=H,
            qw=self.qw.data_ptr(), kw=self.kw.data_ptr(), eps=e.d.eps, cq=s.cq.data_ptr(), frag=int(frag), cache=cache.data_ptr(), gate=L.ptr(gate),
            num_live=L.ptr(b.num_live), x=x.data_ptr(), wp=e.width, state=None if shift is None else shift[i].data_ptr(), state_slot=e.state_slot.data_ptr(), T=T,
            elem=e.elem.code, **self._where(e, b)))
        e._mm(s.cq, self.uq, s.q, T)
        e._heads_mm(s.q, self.uk, s.ql, T, H)
        tiles, n_tiles = b.items(self.tiles)
        self._launch(e, "omni_latent_attn", L.LatentAttn(
            q=s.ql.data_ptr(), cache=cache.data_ptr(), gate=L.ptr(gate), out=s.ol.data_ptr(), tiles=L.ptr(tiles), n_tiles=n_tiles, tile_rows=self.tiles[2], T=T,
            n_decode=b.n_decode, heads=H, rp=self.rp, scale=m.scale, max_keys=b.max_keys, workspace=e.attn_ws.data_ptr(), workspace_bytes=e.attn_ws.numel() * 4,
            elem=e.elem.code, **self._where(e, b)))
        e._heads_mm(s.ol, self.uv, s.v, T, H, out_frag=frag)
        return e._mm(s.v, self.o, s.y, T, f32_out=True)


def rotation_table(rows: int, dims: int, base: float) -> torch.Tensor:
    """fp32 [rows, dims / 2, 2]: cos and sin of position * base^(-2 i / dims)."""
    f = torch.tensor([base ** (-2.0 * i / dims) for i in range(dims // 2)], dtype=torch.float64)
    a = torch.arange(rows, dtype=torch.float64)[:, None] * f
    return torch.stack([a.cos(), a.sin()], -1).to(torch.float32)


class WindowMixer(Mixer):
    def __init__(self, eng, i: int, m: WindowAttentionSpec, w: dict):
        super().__init__(m)
        elem, dev, W, H, G = eng.elem, eng.device, eng.width, m.heads, m.kv_heads
        self.dp, self.vp, self.own = r32(m.dim), r32(m.vdim), m.kv_from is None
        parts = [pad_head_rows(w["q"], H, m.dim, self.dp, W)]
        if self.own:
            parts += [pad_head_rows(w["k"], G, m.dim, self.dp, W), pad_head_rows(w["v"], G, m.vdim, self.vp, W)]
        if m.out_gate:
            parts.append(pad_head_rows(w["g"], H, m.vdim, self.vp, W))
        self.down = Matrix(torch.cat(parts), elem, dev)
        self.qw = eng.up(pad_heads(w["q.norm"], H, m.dim, self.dp)) if m.qk_norm else None
        self.kw = eng.up(pad_heads(w["k.norm"], G, m.dim, self.dp)) if m.qk_norm and self.own else None
        self.sink = w["sink"].to(device=dev, dtype=torch.float32).contiguous() if m.sink else None
        self.o = Matrix(pad_head_cols(w["o"], H, m.vdim, self.vp, W), elem, dev)
        self.rot = eng.shared(("rotation", m.rot_dims, m.rot_base), lambda: rotation_table(eng.d.max_model_len, m.rot_dims, m.rot_base).to(dev)) if m.rot_dims else None
        self.tiles = ("tiles", H // G, eng.lib.omni_window_attn_tile_rows(self.dp, self.vp))
        self.work = (self.tiles,)

    def matrices(self):
        return [self.down, self.o]

    def cache(self, eng, num_blocks, block_size):
        if not self.own:
            return ()
        z = lambda n: torch.zeros(num_blocks, self.spec.kv_heads, block_size, n, dtype=eng.elem.torch, device=eng.device)  # noqa: E731
        return z(self.dp), z(self.vp)

    def workspace_bytes(self, eng, rows):
        return eng.lib.omni_window_attn_workspace_bytes(rows, self.spec.heads, self.vp)

    def needs(self):
        H = self.spec.heads
        return {"proj": (self.down.N, torch.float32, "slabs"), "q": (H * self.dp, "elem", "rows"), "gate": (H * self.vp, "elem", "rows"), "v": (H * self.vp, "elem", "tiles")}

    def run(self, e, b, i, s, x, frag):
        m = self.spec
        T, H = b.T, m.heads
        kc, vc = e.kv_caches[e.d.kv_owner(i)]
        slabs = e._mm(s.h, self.down, s.proj, T, f32_out=True)
        gate = s.gate if m.out_gate else None
        self._launch(e, "omni_qkv_write", L.QkvWrite(
            proj=s.proj.data_ptr(), slabs=slabs, slab_stride=T * self.down.N, ld=self.down.N, heads=H, kv_heads=m.kv_heads, dim=m.dim, dp=self.dp, vp=self.vp,
            qw=L.ptr(self.qw), kw=L.ptr(self.kw), eps=e.d.eps, rot=L.ptr(self.rot), rot_dims=m.rot_dims, rot_rows=0 if self.rot is None else self.rot.shape[0],
            q=s.q.data_ptr(), kc=kc.data_ptr() if self.own else None, vc=vc.data_ptr() if self.own else None, gate=L.ptr(gate), num_live=L.ptr(b.num_live), T=T,
            elem=e.elem.code, **self._where(e, b)))
        tiles, n_tiles = b.items(self.tiles)
        self._launch(e, "omni_window_attn", L.WindowAttn(
            q=s.q.data_ptr(), kc=kc.data_ptr(), vc=vc.data_ptr(), gate=L.ptr(gate), sink=L.ptr(self.sink), out=s.v.data_ptr(), frag=int(frag), tiles=L.ptr(tiles),
            n_tiles=n_tiles, tile_rows=self.tiles[2], T=T, n_decode=b.n_decode, heads=H, kv_heads=m.kv_heads, dp=self.dp, vp=self.vp, scale=m.scale, window=m.window or 0,
            max_keys=b.max_keys, workspace=e.attn_ws.data_ptr(), workspace_bytes=e.attn_ws.numel() * 4, elem=e.elem.code, **self._where(e, b)))
        return e._mm(s.v, self.o, s.y, T, f32_out=True)


class DecayMixer(Mixer):
    def __init__(self, eng, i: int, m: DecayRecurrenceSpec, w: dict):
        super().__init__(m)
        elem, dev, W, H = eng.elem, eng.device, eng.width, m.heads
        self.dp, self.vp = r32(m.dim), r32(m.vdim)
        self.down = Matrix(torch.cat([pad_head_rows(w["q"], H, m.dim, self.dp, W), pad_head_rows(w["k"], H, m.dim, self.dp, W),
                                      pad_head_rows(w["v"], H, m.vdim, self.vp, W), pad_head_rows(w["g"], H, m.vdim, self.vp, W)]), elem, dev)
        self.norm = eng.up(pad_heads(w["norm"], H, m.vdim, self.vp))
        self.o = Matrix(pad_head_cols(w["o"], H, m.vdim, self.vp, W), elem, dev)
        self.decay = torch.tensor(m.decay, dtype=torch.float32, device=dev)
        self.log2_decay = torch.tensor([math.log2(f) for f in m.decay], dtype=torch.float32, device=dev)
        self.chunked = elem.code == 0 and max(self.dp, self.vp) <= L.REC_MAX_DIM
        self.work = (("chunks",), ("segs",), ("runs",))

    def matrices(self):
        return [self.down, self.o]

    def state(self, eng, slots):
        return torch.zeros(slots, self.spec.heads, self.dp, self.vp, dtype=torch.float32, device=eng.device)

    def needs(self):
        n = self.spec.heads * self.vp
        return {"proj": (self.down.N, torch.float32, "slabs"), "rec": (n, torch.float32, "rows"), "v": (n, "elem", "tiles")}

    def run(self, e, b, i, s, x, frag):
        m = self.spec
        T, H, ld, n = b.T, m.heads, self.down.N, m.heads * self.vp
        gcol = H * (2 * self.dp + self.vp)
        wide = e.elem.code == 0 and not frag              # prompts: activations in the product's epilogue, bf16 rows
        if wide:
            proj = s.proj.view(torch.bfloat16)
            e._tile(s.h, self.down, proj, T, act=L.TILE_ACT_SILU_SIGMOID, act_cols=gcol)
            slabs, gate = 0, proj.data_ptr() + 2 * gcol
        else:
            slabs = e._mm(s.h, self.down, s.proj, T, f32_out=True)
            gate = s.proj.data_ptr() + 4 * gcol
        a = L.DecayRec(proj=s.proj.data_ptr(), slabs=slabs, slab_stride=T * ld, ld=ld, heads=H, dp=self.dp, vp=self.vp, decay=self.decay.data_ptr(),
                       log2_decay=self.log2_decay.data_ptr(), state=e.rec_state[i].data_ptr(), state_slot=e.state_slot.data_ptr(), row_of_tok=b.row_of_tok.data_ptr(),
                       positions=b.positions.data_ptr(), num_live=L.ptr(b.num_live), n_decode=b.n_decode, out=s.rec.data_ptr())
        if wide and self.chunked:
            (chunks, n_chunks), (segs, n_segs) = b.items(("chunks",)), b.items(("segs",))
            a.chunks, a.n_chunks, a.segs, a.n_segs = L.ptr(chunks), n_chunks, L.ptr(segs), n_segs
            a.chunk_states = e.chunk_states(n_chunks * H * self.dp * self.vp).data_ptr()
        else:
            runs, a.n_runs = b.items(("runs",))
            a.runs = L.ptr(runs)
        self._launch(e, "omni_decay_rec", a)
        self._launch(e, "omni_gated_norm", L.GatedNorm(o=s.rec.data_ptr(), w=self.norm.data_ptr(), gate=gate, slabs=slabs, slab_stride=T * ld, ld=ld, n=n, count=H * m.vdim,
                                                    eps=e.d.eps, out=s.v.data_ptr(), frag=int(frag), T=T, elem=e.elem.code))
        return e._mm(s.v, self.o, s.y, T, f32_out=True)


MIXERS = {LatentAttentionSpec: LatentMixer, WindowAttentionSpec: WindowMixer, DecayRecurrenceSpec: DecayMixer}


def make_mixer(eng, i: int, weights: dict) -> Mixer:
    """The mixer of weight-owning layer i; `weights`: the checkpoint's tensors."""
    m, p = eng.d.layers[i].mixer, f"l{i}.mix."
    return MIXERS[type(m)](eng, i, m, {k[len(p):]: t for k, t in weights.items() if k.startswith(p)})


# ---------------------------------------------------------------- what a layer keeps, from its spec alone
def cache_row_widths(d: DecoderDims, i: int, elem_code: int) -> tuple[int, ...]:
    """Padded widths of what layer i caches per token (empty: nothing of its own)."""
    m = d.layers[i].mixer
    if isinstance(m, LatentAttentionSpec):
        return (latent_width(m.kv_rank, elem_code),)
    if isinstance(m, WindowAttentionSpec) and m.kv_from is None:
        return (m.kv_heads * r32(m.dim), m.kv_heads * r32(m.vdim))
    return ()


def cache_traffic(d: DecoderDims, i: int, ctx: int) -> tuple[int, int]:
    """(cache elements read, written) by layer i for one token that sees `ctx` tokens."""
    m = d.layers[i].mixer
    if isinstance(m, LatentAttentionSpec):
        return ctx * m.kv_rank, m.kv_rank
    if isinstance(m, WindowAttentionSpec):
        n = m.kv_heads * (m.dim + m.vdim)
        return min(ctx, m.window or ctx) * n, n if m.kv_from is None else 0
    return 0, 0


def state_bytes(d: DecoderDims, i: int) -> int:
    """fp32 recurrent state of one sequence in layer i."""
    m = d.layers[i].mixer
    return 4 * m.heads * m.dim * m.vdim if isinstance(m, DecayRecurrenceSpec) else 0
