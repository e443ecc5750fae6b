"""DecoderEngine: device-resident weights, paged latent cache, per-sequence state and the step function of decoder-only language models.

One forward serves every step: a batch is T tokens, sequence after sequence, the single-token sequences (decoded tokens) first; per layer

  stream_rows    x += g * y / rms(y) of the sublayer before, token shift against the previous token (state for a batch's first one) -> h
  GEMM           [W_dq ; W_dkv ; W_g] h -> fp32: the three products of h are one
  latent_write   both latent norms, the new latent into the cache, gates, the shift state of each sequence's last token
  GEMM, head     q = W_uq c_q, then q_h W_uk,h: queries in the latent space, so that the cache row is key AND value of every head
  latent_attn    causal softmax over the cache (fp32 scores and weights), gate applied to the normalised sum
  head, GEMM     W_uv,h per head, W_o -> y (fp32)
  stream_rows    x += g * y / rms(y) -> bf16 x;  GEMM with xIELU in its epilogue;  GEMM -> y (fp32)

The residual stream, norms, gates, scores and state are fp32; matrix operands are bf16 (``dtype="bfloat16"``) or everything is fp32
(``dtype="float32"``).  GEMMs of up to 64 tokens stream fragment-major weights (omni_gemm_stream), larger ones run omni_gemm_tile on the
SAME bytes.  Every width is padded to a multiple of 32 with zero weights at load, so no size is special.
"""
from __future__ import annotations

import ctypes as C
from dataclasses import dataclass

import torch

from . import _lib as L
from . import ops
from .decoder_config import DecoderDims
from .engine import frag_shuffle

SKINNY = 64            # most tokens of the weight-streaming GEMMs
HEAD_TILE = 512        # from this many tokens on the per-head products run on omni_gemm_tile's column groups


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
    out = torch.zeros(rows, cols, dtype=w.dtype)
    out[:w.shape[0], :w.shape[1]] = w
    return out


def pad1(v: torch.Tensor, n: int) -> torch.Tensor:
    out = torch.zeros(n, dtype=v.dtype)
    out[:v.shape[0]] = v
    return out


class _Matrix:
    """One weight [N, K] (or [heads, N, K]) of a layer, padded, on the device: fragment-major in bf16, row-major in fp32."""

    def __init__(self, w: torch.Tensor, elem: Elem, device):
        w = w.to(device=device, dtype=elem.torch).contiguous()
        self.t = frag_shuffle(w) if elem.code == 0 else w
        self.N, self.K = w.shape[-2:]


class _Layer:
    """Device tensors of one weight-owning layer."""

    def __init__(self, d: DecoderDims, i: int, w: dict, elem: Elem, device):
        s, p = d.layers[i], f"l{i}."
        m = s.mixer
        H, W = m.heads, r32(d.hidden)
        self.qp, self.rp, self.dp, self.vp = r32(m.q_rank), latent_width(m.kv_rank, elem.code), r32(m.dim), r32(m.vdim)
        up = lambda t: t.to(device=device, dtype=elem.torch).contiguous()  # noqa: E731
        parts = [pad2(w[p + "mix.dq"], self.qp, W), pad2(w[p + "mix.dkv"], self.rp, W)]
        if m.out_gate:
            parts.append(pad2(w[p + "mix.g"], r32(H), W))
        self.down = _Matrix(torch.cat(parts), elem, device)
        self.qw, self.kw = up(pad1(w[p + "mix.dq.norm"], self.qp)), up(pad1(w[p + "mix.dkv.norm"], self.rp))
        uq = torch.stack([pad2(h, self.dp, self.qp) for h in w[p + "mix.uq"].reshape(H, m.dim, m.q_rank)])
        self.uq = _Matrix(uq.reshape(H * self.dp, self.qp), elem, device)
        # per head: queries into the latent space (the transpose of W_uk) and latents to values
        self.uk = _Matrix(torch.stack([pad2(h.T, self.rp, self.dp) for h in w[p + "mix.uk"].reshape(H, m.dim, m.kv_rank)]), elem, device)
        self.uv = _Matrix(torch.stack([pad2(h, self.vp, self.rp) for h in w[p + "mix.uv"].reshape(H, m.vdim, m.kv_rank)]), elem, device)
        o = torch.stack([pad2(h, W, self.vp) for h in w[p + "mix.o"].reshape(d.hidden, H, m.vdim).permute(1, 0, 2)], 1)
        self.o = _Matrix(o.reshape(W, H * self.vp), elem, device)
        self.mu = up(pad1(w[p + "shift"], W))
        self.gain1 = float(w[p + "norm1"])
        if s.mlp is not None:
            F = r32(s.mlp.ff)
            self.gain2 = float(w[p + "norm2"])
            self.up, self.dn = _Matrix(pad2(w[p + "mlp.up"], F, W), elem, device), _Matrix(pad2(w[p + "mlp.down"], W, F), elem, device)
            ap, an = torch.nn.functional.softplus(w[p + "mlp.act"].double()).tolist()
            self.act = (ap, 0.5 + an)


class _Scratch:
    """Activations of one forward at a capacity of `rows` tokens; every layer shares them."""

    def __init__(self, eng: "DecoderEngine", rows: int):
        self.rows = rows
        r16 = (rows + 15) // 16 * 16                       # fragment-major operands come in whole 16-row tiles
        dev, E = eng.device, eng.elem.torch
        ls = [eng.layer_w[eng.d.owner(i)] for i in range(eng.d.num_layers)]
        hs = [s.mixer.heads for s in eng.d.layers]
        W = eng.width
        z = lambda n, dt: torch.zeros(n, dtype=dt, device=dev)  # noqa: E731
        self.x = (z(rows * W, torch.float32), z(rows * W, torch.float32))
        # products that leave as partial sums (omni_gemm_stream): as many slabs as up to SKINNY rows may take
        slabs = lambda n: max(rows, min(rows, SKINNY) * L.STREAM_MAX_SPLITS) * n  # noqa: E731
        self.y, self.h = z(slabs(W), torch.float32), z(r16 * W, E)
        self.proj = z(slabs(max(l.down.N for l in ls)), torch.float32)
        self.cq = z(r16 * max(l.qp for l in ls), E)
        self.q = z(rows * max(h * l.dp for h, l in zip(hs, ls)), E)
        self.ql = z(rows * max(h * l.rp for h, l in zip(hs, ls)), E)
        self.ol = torch.zeros_like(self.ql)
        self.v = z(r16 * max(h * l.vp for h, l in zip(hs, ls)), E)
        self.gate = z(rows * max(hs), torch.float32)
        self.act = z(r16 * max([r32(s.mlp.ff) for s in eng.d.layers if s.mlp is not None] or [32]), E)
        self.hn = z(r16 * W, E)


@dataclass
class Batch:
    """One forward's tokens (device tensors).  Tokens [0, n_decode) are single-token sequences; `tiles` covers the rest per (head count, rows of a work item)."""
    T: int
    n_decode: int
    ids: torch.Tensor                   # int32 [T]
    row_of_tok: torch.Tensor            # int32 [T]
    positions: torch.Tensor             # int32 [T]
    tiles: dict[tuple, torch.Tensor]    # (heads, tile rows) -> int32 [2 n]
    max_keys: int                       # most keys a decode token sees
    num_live: torch.Tensor | None = None


def attention_tiles(seg_starts: list[int], seg_lens: list[int], heads: int, tile_rows: int) -> list[tuple[int, int]]:
    """Work items of the prompt attention: runs of up to `tile_rows` query rows (token-major, heads inside) of ONE sequence.  Longest first: a later
    tile of a prompt sees more keys."""
    out = []
    for s, n in zip(seg_starts, seg_lens):
        lo, hi = s * heads, (s + n) * heads
        out += [(lo - f, f, min(tile_rows, hi - f)) for f in range(lo, hi, tile_rows)]
    return [(f, n) for _, f, n in sorted(out)]


class DecoderEngine:
    def __init__(self, dims: DecoderDims, weights: dict, *, dtype: str = "bfloat16", kv_dtype: str = "auto", num_blocks: int = 1024, block_size: int = 16,
                 max_batch: int = 64, device: str = "cuda:0"):
        if not torch.cuda.is_available():
            raise L.OmniError("DecoderEngine needs an MI355X (torch.cuda unavailable); there is no CPU fallback")
        if dtype not in ELEM:
            raise ValueError(f"dtype {dtype!r}: one of {sorted(ELEM)}")
        self.elem = ELEM[dtype]
        if kv_dtype not in self.elem.kv_names:
            raise ValueError(f"kv_cache_dtype {kv_dtype!r}: the latent cache is kept in the model's dtype ({self.elem.kv_names} for {dtype})")
        if block_size & (block_size - 1):
            raise ValueError(f"block_size {block_size}: a power of two")
        self.lib = L.load_decoder()
        self.d, self.device, self.kv_dtype = dims, torch.device(device), kv_dtype
        self.block_size, self.max_batch = block_size, max_batch
        self.width = r32(dims.hidden)
        self.bt_stride = (dims.max_model_len + block_size - 1) // block_size
        dev, E = self.device, self.elem.torch
        # ---- weights
        self.embed = pad2(weights["embed"], dims.vocab, self.width).to(device=dev, dtype=E)
        self.head = _Matrix(pad2(weights["head"], r32(dims.vocab), self.width), self.elem, dev)
        self.final_gain = float(weights["final.norm"])
        self.layer_w = {i: _Layer(dims, i, weights, self.elem, dev) for i in range(dims.num_layers) if dims.owner(i) == i}
        # per layer: heads and query rows per work item of its prompt attention
        self.tile_kinds = [(s.mixer.heads, self.lib.omni_latent_attn_tile_rows(self.layer_w[dims.owner(i)].rp)) for i, s in enumerate(dims.layers)]
        self._alloc_kv(num_blocks)
        # ---- per-sequence state: what each layer's mixer read at the sequence's last token; slot 0 belongs to no sequence
        self.state_slots = max_batch + 1
        self.state = torch.zeros(dims.num_layers, self.state_slots, self.width, dtype=torch.float32, device=dev)
        # ---- persistent per-row buffers (graph-stable addresses)
        Bm = max_batch
        i32 = dict(dtype=torch.int32, device=dev)
        self.ids_status = torch.zeros(Bm + 4, **i32)        # sampled ids and the step's status words: what the runner copies per step
        self.out_record = self.ids_status
        self.input_ids, self.status = self.ids_status[:Bm], self.ids_status[Bm:]
        self.positions, self.seq_lens, self.steps = torch.zeros(Bm, **i32), torch.ones(Bm, **i32), torch.zeros(Bm, **i32)
        self.block_table = torch.zeros(Bm, self.bt_stride, **i32)
        self.state_slot = torch.zeros(Bm, **i32)
        self.row_ids = torch.arange(Bm, **i32)
        self.num_live = torch.full((1,), Bm, **i32)
        self.seen = torch.zeros(Bm, dims.vocab, dtype=torch.uint8, device=dev)
        self.logits = torch.zeros(Bm, self.head.N, dtype=torch.float32, device=dev)
        self.row_greedy, self.row_top_k, self.row_seed = torch.ones(Bm, **i32), torch.zeros(Bm, **i32), torch.zeros(Bm, **i32)
        f32 = dict(dtype=torch.float32, device=dev)
        self.row_temperature, self.row_top_p, self.row_rep_penalty = torch.ones(Bm, **f32), torch.ones(Bm, **f32), torch.ones(Bm, **f32)
        # ---- scratch: the decode step's own (its addresses are recorded in graphs), and one that grows with the prompts
        self._dec = _Scratch(self, Bm)
        self._any: _Scratch | None = None
        heads = max(s.mixer.heads for s in dims.layers)
        rp = max(l.rp for l in self.layer_w.values())
        nbytes = self.lib.omni_latent_attn_workspace_bytes(Bm, heads, rp)
        self.attn_ws = torch.zeros(nbytes // 4, dtype=torch.float32, device=dev)
        self.persistent_chains = False

    # ------------------------------------------------------------------ cache
    def _alloc_kv(self, num_blocks: int) -> None:
        self.num_blocks = int(num_blocks)
        self.kv_caches = [torch.zeros(self.num_blocks, self.block_size, self.layer_w[self.d.owner(i)].rp, dtype=self.elem.torch, device=self.device)
                          for i in range(self.d.num_layers)]

    def kv_cache_bytes(self) -> int:
        return sum(c.numel() * c.element_size() for c in self.kv_caches)

    def resize_kv_cache(self, num_blocks: int) -> None:
        """Another number of blocks (before any graph capture)."""
        self.kv_caches = None
        torch.cuda.empty_cache()
        self._alloc_kv(num_blocks)

    def profile_run(self, num_tokens: int, batch: int) -> None:
        """The worker's memory probe: a prompt step of `num_tokens` tokens over `batch` rows and a decode step, on the probe cache."""
        batch = max(1, min(batch, self.max_batch))
        per = max(1, min(num_tokens // batch, self.d.max_model_len - 2, (self.num_blocks - 1) // batch * self.block_size - 1))
        need = (per + 1 + self.block_size - 1) // self.block_size
        bt = torch.zeros(self.max_batch, self.bt_stride, dtype=torch.int32)
        for r in range(batch):
            bt[r, :need] = torch.arange(1 + r * need, 1 + (r + 1) * need, dtype=torch.int32)
        self.block_table.copy_(bt)
        pos, row = torch.arange(per).repeat(batch), torch.arange(batch).repeat_interleave(per)
        b = self.make_batch(torch.zeros(batch * per, dtype=torch.int32), row, pos, [per] * batch)
        self.forward(b, sel=torch.arange(batch, dtype=torch.int32, device=self.device))
        self.positions[:batch] = per
        self.decode_step(batch)
        torch.cuda.synchronize(self.device)
        self.seq_lens.fill_(1)
        for t in (self.positions, self.steps, self.seen, self.block_table, self.input_ids):
            t.zero_()

    # ------------------------------------------------------------------ sampling parameters (one request's SamplingParams per row)
    ROW_KEYS = ("greedy", "temperature", "top_k", "top_p", "rep_penalty", "seed")
    MAX_SAMPLED_VOCAB = 8192           # csrc/sampler_body.cuh SMP_MAXV

    def set_row_sampling(self, row: int, *, greedy, temperature, top_k, top_p, rep_penalty, seed) -> None:
        if not greedy and not temperature > 0.0:
            raise ValueError("temperature must be > 0 when sampling")
        seed = int(seed) & 0xFFFFFFFF
        for k, v in (("greedy", int(bool(greedy))), ("temperature", temperature if temperature > 0 else 1.0), ("top_k", top_k), ("top_p", top_p),
                     ("rep_penalty", rep_penalty), ("seed", seed - (1 << 32) if seed >= (1 << 31) else seed)):
            getattr(self, "row_" + k)[row] = v

    # ------------------------------------------------------------------ products
    def _mm(self, x: torch.Tensor, w: _Matrix, out: torch.Tensor, T: int, *, f32_out: bool = False, one: bool = False, act=None, out_frag: bool = False) -> int:
        """out [T, N] = (xIELU of) x . w^T.  x: fragment-major when T <= SKINNY and bf16 (its producer wrote it so), else row-major.  Returns how
        many partial sums [T, N] an fp32 output consists of (its consumer adds them up; one: a single one)."""
        st, lib = L.current_stream(), self.lib
        a, b = act or (0.0, 0.0)
        if self.elem.code == 1:
            L.check(lib.omni_gemm_f32(x.data_ptr(), w.K, 0, w.t.data_ptr(), 0, out.data_ptr(), w.N, 0, T, w.N, w.K, 1, int(act is not None), a, b, st),
                    "omni_gemm_f32", lib)
        elif T <= SKINNY:
            kind = L.STREAM_F32 if f32_out else (L.STREAM_BF16 if act is None else L.STREAM_XIELU)
            L.check(lib.omni_gemm_stream(x.data_ptr(), w.t.data_ptr(), out.data_ptr(), T, w.N, w.K, kind, int(one), a, b, int(out_frag), st), "omni_gemm_stream", lib)
            return lib.omni_gemm_stream_splits(T, w.N, w.K) if f32_out and not one else 1
        else:
            o = out[:T * w.N].view(T, w.N)
            ops.gemm_tile(x[:T * w.K].view(T, w.K), w.t, act=L.TILE_ACT_NONE if act is None else L.TILE_ACT_XIELU, act_params=(a, b),
                          want="f" if f32_out else "b", lib=lib, **({"out_f32": o} if f32_out else {"out": o}))
        return 1

    def _heads_mm(self, x: torch.Tensor, w: _Matrix, out: torch.Tensor, T: int, heads: int, out_frag: bool = False) -> None:
        """out[t, h] = x[t, h] . w[h]^T."""
        st, lib = L.current_stream(), self.lib
        if self.elem.code == 1:
            L.check(lib.omni_gemm_f32(x.data_ptr(), heads * w.K, w.K, w.t.data_ptr(), w.N * w.K, out.data_ptr(), heads * w.N, w.N, T, w.N, w.K, heads, 0,
                                      0.0, 0.0, st), "omni_gemm_f32", lib)
        elif T < HEAD_TILE or heads == 1:
            L.check(lib.omni_head_gemm(x.data_ptr(), w.t.data_ptr(), out.data_ptr(), T, heads, w.N, w.K, int(out_frag), st), "omni_head_gemm", lib)
        else:
            ops.gemm_tile(x[:T * heads * w.K].view(T, heads * w.K), w.t, groups=heads, group_cols=True, out=out[:T * heads * w.N].view(T, heads * w.N), lib=lib)

    def _rows(self, **kw) -> None:
        a = L.StreamRows(width=self.d.hidden, wp=self.width, eps=self.d.eps, elem=self.elem.code)
        for k, v in kw.items():
            setattr(a, k, L.ptr(v) if isinstance(v, torch.Tensor) else v)
        L.check(self.lib.omni_stream_rows_run(C.byref(a), L.current_stream()), "omni_stream_rows", self.lib)

    # ------------------------------------------------------------------ forward
    def make_batch(self, ids: torch.Tensor, row_of_tok, positions, seg_lens: list[int], *, n_decode: int = 0, max_keys: int = 0, ids_device=None) -> Batch:
        """A batch from host arrays: tokens [0, n_decode) single-token sequences, then segments of `seg_lens` tokens.  One upload."""
        T = len(row_of_tok)
        kinds = sorted(set(self.tile_kinds)) if T > n_decode else []
        starts, o = [], n_decode
        for n in seg_lens:
            starts.append(o)
            o += n
        assert o == T, (o, T)
        tl = {k: attention_tiles(starts, seg_lens, *k) for k in kinds}
        flat = [torch.as_tensor(ids, dtype=torch.int32), torch.as_tensor(row_of_tok, dtype=torch.int32), torch.as_tensor(positions, dtype=torch.int32)]
        flat += [torch.tensor(tl[k], dtype=torch.int32).reshape(-1) for k in kinds]
        buf = torch.cat(flat).pin_memory().to(self.device, non_blocking=True)
        tiles, o = {}, 3 * T
        for k in kinds:
            n = 2 * len(tl[k])
            tiles[k] = buf[o:o + n]
            o += n
        return Batch(T, n_decode, buf[:T] if ids_device is None else ids_device, buf[T:2 * T], buf[2 * T:3 * T], tiles, max_keys)

    def _scratch(self, T: int) -> _Scratch:
        if self._any is None or self._any.rows < T:
            self._any = None
            self._any = _Scratch(self, max(T, 256) if T <= 256 else (T + 1023) // 1024 * 1024)
        return self._any

    def _mixer(self, b: Batch, i: int, s: _Scratch, x: torch.Tensor, frag: bool) -> int:
        """s.h -> s.y (returns its partial sums)"""
        m, w, lib, st = self.d.layers[i].mixer, self.layer_w[self.d.owner(i)], self.lib, L.current_stream()
        T, H = b.T, m.heads
        slabs = self._mm(s.h, w.down, s.proj, T, f32_out=True)
        gate = s.gate if m.out_gate else None
        a = L.LatentWrite(proj=s.proj.data_ptr(), slabs=slabs, slab_stride=T * w.down.N, ld=w.down.N, q_rank=m.q_rank, qp=w.qp, kv_rank=m.kv_rank, rp=w.rp, heads=H, qw=w.qw.data_ptr(),
                          kw=w.kw.data_ptr(), eps=self.d.eps, cq=s.cq.data_ptr(), frag=int(frag), cache=self.kv_caches[i].data_ptr(), gate=L.ptr(gate),
                          block_table=self.block_table.data_ptr(), bt_stride=self.bt_stride, block_size=self.block_size, row_of_tok=b.row_of_tok.data_ptr(),
                          positions=b.positions.data_ptr(), num_live=L.ptr(b.num_live), x=x.data_ptr(), wp=self.width, state=self.state[i].data_ptr(),
                          state_slot=self.state_slot.data_ptr(), T=T, elem=self.elem.code)
        L.check(lib.omni_latent_write_run(C.byref(a), st), "omni_latent_write", lib)
        self._mm(s.cq, w.uq, s.q, T)
        self._heads_mm(s.q, w.uk, s.ql, T, H)
        tiles = b.tiles.get(self.tile_kinds[i])
        a = L.LatentAttn(q=s.ql.data_ptr(), cache=self.kv_caches[i].data_ptr(), gate=L.ptr(gate), out=s.ol.data_ptr(), block_table=self.block_table.data_ptr(),
                         bt_stride=self.bt_stride, block_size=self.block_size, row_of_tok=b.row_of_tok.data_ptr(), positions=b.positions.data_ptr(),
                         tiles=L.ptr(tiles), n_tiles=0 if tiles is None else tiles.numel() // 2, tile_rows=self.tile_kinds[i][1], T=T, n_decode=b.n_decode, heads=H, rp=w.rp, scale=m.scale,
                         max_keys=b.max_keys, workspace=self.attn_ws.data_ptr(), workspace_bytes=self.attn_ws.numel() * 4, elem=self.elem.code)
        L.check(lib.omni_latent_attn_run(C.byref(a), st), "omni_latent_attn", lib)
        self._heads_mm(s.ol, w.uv, s.v, T, H, out_frag=frag)
        return self._mm(s.v, w.o, s.y, T, f32_out=True)

    def forward(self, b: Batch, *, sel: torch.Tensor | None = None, logits: torch.Tensor | None = None, scratch: _Scratch | None = None,
                trail: list | None = None) -> torch.Tensor | None:
        """All layers over a batch; logits fp32 [len(sel), padded vocab] of the selected tokens (sel None: of every token; sel empty: none).
        trail: gets the residual stream behind every layer (diagnostics)."""
        d, s = self.d, scratch or self._scratch(b.T)
        T = b.T
        frag = self.elem.code == 0 and T <= SKINNY
        lw = lambda i: self.layer_w[d.owner(i)]  # noqa: E731
        where = dict(row_of_tok=b.row_of_tok, positions=b.positions, state_slot=self.state_slot, rows=T)
        k = 0
        self._rows(ids=b.ids, table=self.embed, vocab=d.vocab, mu=lw(0).mu, state=self.state[0], x_out=s.x[k], h_out=s.h, frag=int(frag), **where)
        for i in range(d.num_layers):
            w = lw(i)
            ny, gain = self._mixer(b, i, s, s.x[k], frag), w.gain1
            if d.layers[i].mlp is not None:
                self._rows(x_in=s.x[k], y=s.y, y_slabs=ny, y_stride=T * self.width, gain=gain, x_out=s.x[k ^ 1], h_out=s.h, frag=int(frag), rows=T)
                k ^= 1
                self._mm(s.h, w.up, s.act, T, act=w.act, out_frag=frag)
                ny, gain = self._mm(s.act, w.dn, s.y, T, f32_out=True), w.gain2
            add = dict(x_in=s.x[k], y=s.y, y_slabs=ny, y_stride=T * self.width, gain=gain)
            if trail is not None:
                self._rows(**add, x_out=s.x[k ^ 1], rows=T)
                trail.append(s.x[k ^ 1][:T * self.width].view(T, self.width)[:, :d.hidden].clone())
            if i + 1 < d.num_layers:
                self._rows(**add, mu=lw(i + 1).mu, state=self.state[i + 1], x_out=s.x[k ^ 1], h_out=s.h, frag=int(frag), **where)
                k ^= 1
        n = T if sel is None else sel.numel()
        if n == 0:
            return None
        if n > s.rows:
            raise L.OmniError(f"logits of {n} rows from a batch of {T} tokens")
        nfrag = self.elem.code == 0 and n <= SKINNY
        self._rows(**add, use_final=1, final_gain=self.final_gain, sel=sel, h_out=s.hn, frag=int(nfrag), rows=n)
        if logits is None:
            logits = torch.empty(n, self.head.N, dtype=torch.float32, device=self.device)
        self._mm(s.hn, self.head, logits.view(-1), n, f32_out=True, one=True)
        return logits

    def sample_rows_in_place(self, B: int, num_live: torch.Tensor) -> None:
        """Rows [0, B): next id from self.logits into input_ids, repetition bitmap, step counter, position and length advanced."""
        rs = L.RowSampling(*[getattr(self, "row_" + k).data_ptr() for k in self.ROW_KEYS])
        L.check(self.lib.omni_sample_step(self.logits.data_ptr(), self.logits.stride(0), B, self.d.vocab, C.byref(rs), self.seen.data_ptr(), self.steps.data_ptr(),
                                          self.input_ids.data_ptr(), self.positions.data_ptr(), self.seq_lens.data_ptr(), num_live.data_ptr(),
                                          L.current_stream()), "omni_sample_step", self.lib)

    def decode_step(self, B: int, advance: bool = True) -> None:
        """One decode step of rows [0, B) from the persistent buffers (capturable): layers, logits, sampler, counters."""
        b = Batch(B, B, self.input_ids, self.row_ids, self.positions, {}, self.d.max_model_len, self.num_live)
        self.forward(b, logits=self.logits[:B], scratch=self._dec)
        if advance and self.d.vocab <= self.MAX_SAMPLED_VOCAB:
            self.sample_rows_in_place(B, self.num_live)

    # ------------------------------------------------------------------ roofline accounting
    def step_bytes(self, ctx_lens) -> dict:
        """Bytes a decode step must move: matrices of every layer run, the head, and the latents read and written."""
        from .weights import decoder_weight_bytes
        es = torch.empty((), dtype=self.elem.torch).element_size()
        per_tok = sum(s.mixer.kv_rank for s in self.d.layers) * es
        w = decoder_weight_bytes(self.d) * es // 2
        return {"weights": w, "kv_read": int(sum(int(c) for c in ctx_lens)) * per_tok, "kv_write": len(ctx_lens) * per_tok,
                "total": w + (int(sum(int(c) for c in ctx_lens)) + len(ctx_lens)) * per_tok}
