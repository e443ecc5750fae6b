"""DecoderEngine: device-resident weights, paged cache, per-sequence state and the step function of decoder-only language models.

One forward serves every step: a batch is T tokens, sequence after sequence, the single-token sequences (decoded tokens) first.  Per layer

  stream_rows    the sublayer before joins the residual stream -- x += g * y / rms(y), or x = w * (alpha x + y) / rms(..) -- and h follows from x
                 (token shift against the previous token, or x itself)
  mixer          h -> y (decoder_mixers.py): joint projection, cache write / state update, attention or recurrence, output projection
  stream_rows, GEMM with its activation in the epilogue, GEMM       the feed-forward -> y (fp32)
  stream_rows, GEMM (gelu * the token's side row), GEMM             the side input, where the model has one -> y (fp32)

Latent attention, as launches:
  GEMM           [W_dq ; W_dkv ; W_g] h -> fp32: the three products of h are one
  latent_write   both latent norms, the new latent into the cache, gates, the shift state of each sequence's last token
  GEMM, head     q = W_uq c_q, then q_h W_uk,h: queries in the latent space, so that the cache row is key AND value of every head
  latent_attn    causal softmax over the cache (fp32 scores and weights), gate applied to the normalised sum
  head, GEMM     W_uv,h per head, W_o -> y (fp32)
Windowed attention:
  GEMM           [W_q ; W_k ; W_v ; W_g] h -> fp32
  qkv_write      norms over whole projections, rotation, keys and values into the cache, the gate
  window_attn    softmax over the window (and the sink), gate applied;   GEMM  W_o -> y (fp32)
Decay recurrence:
  GEMM           [W_q ; W_k ; W_v ; W_g] h -> fp32 (prompts: SiLU / sigmoid in the epilogue, bf16)
  decay_rec      state update and outputs (prompts: chunks);  gated_norm  the norm over all heads, the gate;  GEMM  W_o -> y (fp32)

The residual stream, norms, gates of norms, scores and state are fp32; matrix operands are bf16 (``dtype="bfloat16"``) or everything is fp32
(``dtype="float32"``).  GEMMs of up to 64 tokens stream fragment-major weights (omni_gemm_stream), larger ones run omni_gemm_tile on the
SAME bytes.  Every width is padded to a multiple of 32 with zero weights at load, so no size is special.
"""
from __future__ import annotations

import ctypes as C
from dataclasses import dataclass, field

import torch

from . import _lib as L
from . import ops
from .decoder_config import DecoderDims
from .decoder_mixers import (ELEM, LATENT_WIDTHS, WORK, Elem, Matrix, attention_tiles, cache_traffic, latent_width, make_mixer, pad1, pad2, r32,  # noqa: F401
                             state_bytes)

SKINNY = 64            # most tokens of the weight-streaming GEMMs
HEAD_TILE = 512        # from this many tokens on the per-head products run on omni_gemm_tile's column groups

# a feed-forward's activation in the three products: (omni_gemm_stream kind, omni_gemm_tile act, omni_gemm_f32 act)
MLP_ACTS = {"xielu": (L.STREAM_XIELU, L.TILE_ACT_XIELU, L.ACT_XIELU), "relu2": (L.STREAM_RELU2, L.TILE_ACT_RELU2, L.ACT_RELU2)}


@dataclass
class Act:
    name: str
    params: tuple[float, float] = (0.0, 0.0)


class _Layer:
    """Device tensors of one weight-owning layer."""

    def __init__(self, eng: "DecoderEngine", i: int, w: dict):
        d, elem, dev = eng.d, eng.elem, eng.device
        s, p, W = d.layers[i], f"l{i}.", eng.width
        self.mixer = make_mixer(eng, i, w)
        self.mu = eng.up(pad1(w[p + "shift"], W)) if d.token_shift else None
        self.norm1 = eng.norm_gain(w[p + "norm1"])
        self.mats = self.mixer.matrices()
        if s.mlp is not None:
            F = r32(s.mlp.ff)
            self.norm2 = eng.norm_gain(w[p + "norm2"])
            self.up, self.dn = Matrix(pad2(w[p + "mlp.up"], F, W), elem, dev), Matrix(pad2(w[p + "mlp.down"], W, F), elem, dev)
            self.mats += [self.up, self.dn]
            self.act = Act(s.mlp.act)
            if s.mlp.act == "xielu":
                ap, an = torch.nn.functional.softplus(w[p + "mlp.act"].double()).tolist()
                self.act.params = (ap, 0.5 + an)
        if d.side_dim:
            self.side_gate, self.side_proj = Matrix(pad2(w[p + "side.gate"], eng.side_width, W), elem, dev), Matrix(pad2(w[p + "side.proj"], W, eng.side_width), elem, dev)
            self.side_norm = eng.up(pad1(w[p + "side.norm"], W))
            self.mats += [self.side_gate, self.side_proj]


class _Scratch:
    """Activations of one forward at a capacity of `rows` tokens; every layer shares them."""

    def __init__(self, eng: "DecoderEngine", rows: int):
        self.rows = rows
        r16 = (rows + 15) // 16 * 16                       # fragment-major operands come in whole 16-row tiles
        # products that leave as partial sums (omni_gemm_stream): as many slabs as up to SKINNY rows may take
        count = {"rows": rows, "tiles": r16, "slabs": max(rows, min(rows, SKINNY) * L.STREAM_MAX_SPLITS)}
        W = eng.width
        needs = [{"x0": (W, torch.float32, "rows"), "x1": (W, torch.float32, "rows"), "y": (W, torch.float32, "slabs"), "h": (W, "elem", "tiles"), "hn": (W, "elem", "tiles"),
                  "act": (max([r32(s.mlp.ff) for s in eng.d.layers if s.mlp is not None] + [eng.side_width, 32]), "elem", "tiles")}]
        needs += [l.mixer.needs() for l in eng.layer_w.values()]
        size: dict[str, tuple] = {}
        for n in needs:
            for k, (width, dt, per) in n.items():
                have = size.get(k)
                assert have is None or have[1:] == (dt, per), k
                size[k] = (max(width, have[0] if have else 0), dt, per)
        for k, (width, dt, per) in size.items():
            setattr(self, k, torch.zeros(count[per] * width, dtype=eng.elem.torch if dt == "elem" else dt, device=eng.device))
        self.x = (self.x0, self.x1)


@dataclass
class Batch:
    """One forward's tokens (device tensors).  Tokens [0, n_decode) are single-token sequences; `work` holds the others' work items per kind."""
    T: int
    n_decode: int
    ids: torch.Tensor                   # int32 [T]
    row_of_tok: torch.Tensor            # int32 [T]
    positions: torch.Tensor             # int32 [T]
    max_keys: int                       # most keys a decode token sees
    work: dict[tuple, tuple[torch.Tensor, int]] = field(default_factory=dict)      # work key -> (int32 items, how many)
    num_live: torch.Tensor | None = None

    def items(self, key: tuple) -> tuple[torch.Tensor | None, int]:
        return self.work.get(key, (None, 0))


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
        self._shared: dict = {}
        self._chunk_states: torch.Tensor | None = None
        self.embed = pad2(weights["embed"], dims.vocab, self.width).to(device=dev, dtype=E)
        self.side_width = r32(dims.side_dim) if dims.side_dim else 0
        if dims.side_dim:                                   # [vocab, layers, padded]: a layer's slice is a column range
            t = weights["side.embed"].reshape(dims.vocab * dims.num_layers, dims.side_dim)
            self.side_embed = pad2(t, t.shape[0], self.side_width).reshape(dims.vocab, dims.num_layers * self.side_width).to(device=dev, dtype=E)
        self.head = Matrix(pad2(weights["head"], r32(dims.vocab), self.width), self.elem, dev)
        self.final_norm = self.norm_gain(weights["final.norm"])
        self.layer_w = {i: _Layer(self, i, weights) for i in range(dims.num_layers) if dims.owner(i) == i}
        self.mixers = [self.layer_w[dims.owner(i)].mixer for i in range(dims.num_layers)]
        self.work_keys = sorted({k for m in self.mixers for k in m.work})
        self._alloc_kv(num_blocks)
        # ---- per-sequence state, slot 0 of no sequence: what each layer's mixer read at the sequence's last token, and the mixers' own
        self.state_slots = max_batch + 1
        self.shift_state = torch.zeros(dims.num_layers, self.state_slots, self.width, dtype=torch.float32, device=dev) if dims.token_shift else None
        self.rec_state = [m.state(self, self.state_slots) for m in self.mixers]
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
        self.attn_ws = torch.zeros(max(m.workspace_bytes(self, Bm) for m in self.mixers) // 4 + 1, dtype=torch.float32, device=dev)
        self.persistent_chains = False

    # ------------------------------------------------------------------ tensors
    def up(self, t: torch.Tensor) -> torch.Tensor:
        """A vector of weights in the model's element type."""
        return t.to(device=self.device, dtype=self.elem.torch).contiguous()

    def norm_gain(self, t: torch.Tensor):
        """A norm's weight: one number, or a padded vector."""
        return float(t) if t.dim() == 0 else self.up(pad1(t, self.width))

    def shared(self, key: tuple, make) -> torch.Tensor:
        """A table that several layers read."""
        if key not in self._shared:
            self._shared[key] = make()
        return self._shared[key]

    def chunk_states(self, elements: int) -> torch.Tensor:
        """Scratch of the chunked recurrence, shared by the layers (prompt steps only: it grows)."""
        if self._chunk_states is None or self._chunk_states.numel() < elements:
            self._chunk_states = None
            self._chunk_states = torch.empty(elements, dtype=torch.float32, device=self.device)
        return self._chunk_states

    # ------------------------------------------------------------------ cache
    def _alloc_kv(self, num_blocks: int) -> None:
        self.num_blocks = int(num_blocks)
        self.kv_caches = [m.cache(self, self.num_blocks, self.block_size) for m in self.mixers]

    def kv_cache_bytes(self) -> int:
        return sum(c.numel() * c.element_size() for layer in self.kv_caches for c in layer)

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
    def _mm(self, x: torch.Tensor, w: Matrix, out: torch.Tensor, T: int, *, f32_out: bool = False, one: bool = False, act: Act | None = None, out_frag: bool = False) -> int:
        """out [T, N] = act(x . w^T).  x: fragment-major when T <= SKINNY and bf16 (its producer wrote it so), else row-major.  Returns how
        many partial sums [T, N] an fp32 output consists of (its consumer adds them up; one: a single one)."""
        st, lib = L.current_stream(), self.lib
        a, b = act.params if act else (0.0, 0.0)
        stream, tile, plain = MLP_ACTS[act.name] if act else (L.STREAM_BF16, L.TILE_ACT_NONE, L.ACT_NONE)
        if self.elem.code == 1:
            L.check(lib.omni_gemm_f32(x.data_ptr(), w.K, 0, w.t.data_ptr(), 0, out.data_ptr(), w.N, 0, T, w.N, w.K, 1, plain, a, b, st), "omni_gemm_f32", lib)
        elif T <= SKINNY:
            kind = L.STREAM_F32 if f32_out else stream
            L.check(lib.omni_gemm_stream(x.data_ptr(), w.t.data_ptr(), out.data_ptr(), T, w.N, w.K, kind, int(one), a, b, int(out_frag), st), "omni_gemm_stream", lib)
            return lib.omni_gemm_stream_splits(T, w.N, w.K) if f32_out and not one else 1
        else:
            self._tile(x, w, out, T, f32_out=f32_out, act=tile, act_params=(a, b))
        return 1

    def _tile(self, x: torch.Tensor, w: Matrix, out: torch.Tensor, T: int, *, f32_out: bool = False, **kw) -> None:
        """omni_gemm_tile on row-major rows."""
        o = out[:T * w.N].view(T, w.N)
        ops.gemm_tile(x[:T * w.K].view(T, w.K), w.t, want="f" if f32_out else "b", lib=self.lib, **({"out_f32": o} if f32_out else {"out": o}), **kw)

    def _mm_rows(self, x: torch.Tensor, w: Matrix, out: torch.Tensor, T: int, table: L.RowTable, out_frag: bool) -> None:
        """out [T, N] = gelu_tanh(x . w^T) * the tokens' rows of a table."""
        st, lib = L.current_stream(), self.lib
        if self.elem.code == 1:
            L.check(lib.omni_gemm_f32_rows(x.data_ptr(), w.K, w.t.data_ptr(), out.data_ptr(), w.N, T, w.N, w.K, C.byref(table), st), "omni_gemm_f32_rows", lib)
        elif T <= SKINNY:
            L.check(lib.omni_gemm_stream_rows(x.data_ptr(), w.t.data_ptr(), out.data_ptr(), T, w.N, w.K, C.byref(table), int(out_frag), st), "omni_gemm_stream_rows", lib)
        else:
            self._tile(x, w, out, T, act=L.TILE_ACT_GELU_MUL, mul=table)

    def _heads_mm(self, x: torch.Tensor, w: Matrix, out: torch.Tensor, T: int, heads: int, out_frag: bool = False) -> None:
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
        keys = self.work_keys if T > n_decode else []
        starts, o = [], n_decode
        for n in seg_lens:
            starts.append(o)
            o += n
        assert o == T, (o, T)
        flat = [torch.as_tensor(ids, dtype=torch.int32), torch.as_tensor(row_of_tok, dtype=torch.int32), torch.as_tensor(positions, dtype=torch.int32)]
        made = {k: WORK[k[0]](starts, seg_lens, *k[1:]) for k in keys}
        flat += [torch.tensor(made[k], dtype=torch.int32).reshape(-1) for k in keys]
        buf = torch.cat(flat).pin_memory().to(self.device, non_blocking=True)
        work, o = {}, 3 * T
        for k, t in zip(keys, flat[3:]):
            work[k] = (buf[o:o + t.numel()], len(made[k]))
            o += t.numel()
        return Batch(T, n_decode, buf[:T] if ids_device is None else ids_device, buf[T:2 * T], buf[2 * T:3 * T], max_keys, work)

    def _scratch(self, T: int) -> _Scratch:
        if self._any is None or self._any.rows < T:
            self._any = None
            self._any = _Scratch(self, max(T, 256) if T <= 256 else (T + 1023) // 1024 * 1024)
        return self._any

    def _join(self, k: int, s: _Scratch, ny: int, T: int, gain) -> dict:
        """stream_rows arguments that let the sublayer output s.y (ny partial sums) join the stream s.x[k] through its norm."""
        add = dict(x_in=s.x[k], y=s.y, y_slabs=ny, y_stride=T * self.width)
        if self.d.norm == "post":
            return dict(add, post=1, alpha=self.d.alpha, y_w=gain)
        return dict(add, gain=gain)

    def forward(self, b: Batch, *, sel: torch.Tensor | None = None, logits: torch.Tensor | None = None, scratch: _Scratch | None = None,
                trail: list | None = None) -> torch.Tensor | None:
        """All layers over a batch; logits fp32 [len(sel), padded vocab] of the selected tokens (sel None: of every token; sel empty: none).
        trail: gets the residual stream behind every layer (diagnostics)."""
        d, s = self.d, scratch or self._scratch(b.T)
        T = b.T
        frag = self.elem.code == 0 and T <= SKINNY
        k = 0

        def operand(i: int | None, **source) -> None:
            """The stream's new rows from `source`, and h of them: layer i's mixer input, or (None) the rows themselves."""
            nonlocal k
            if "x_in" in source:
                k ^= 1
            if i is not None and d.token_shift:
                source.update(mu=self.layer_w[d.owner(i)].mu, state=self.shift_state[i], row_of_tok=b.row_of_tok, positions=b.positions, state_slot=self.state_slot)
            self._rows(**source, x_out=s.x[k], h_out=s.h, frag=int(frag), rows=T)

        operand(0, ids=b.ids, table=self.embed, vocab=d.vocab, table_scale=d.embed_scale)
        for i in range(d.num_layers):
            w = self.layer_w[d.owner(i)]
            add = self._join(k, s, w.mixer.run(self, b, i, s, s.x[k], frag), T, w.norm1)
            if d.layers[i].mlp is not None:
                operand(None, **add)
                self._mm(s.h, w.up, s.act, T, act=w.act, out_frag=frag)
                add = self._join(k, s, self._mm(s.act, w.dn, s.y, T, f32_out=True), T, w.norm2)
            if d.side_dim:
                operand(None, **add)
                table = L.RowTable(self.side_embed[:, i * self.side_width:].data_ptr(), b.ids.data_ptr(), d.vocab, self.side_embed.shape[1])
                self._mm_rows(s.h, w.side_gate, s.act, T, table, frag)
                ny = self._mm(s.act, w.side_proj, s.y, T, f32_out=True)
                add = dict(x_in=s.x[k], y=s.y, y_slabs=ny, y_stride=T * self.width, y_w=w.side_norm)
            if trail is not None:
                self._rows(**add, x_out=s.x[k ^ 1], rows=T)
                trail.append(s.x[k ^ 1][:T * self.width].view(T, self.width)[:, :d.hidden].clone())
            if i + 1 < d.num_layers:
                operand(i + 1, **add)
        n = T if sel is None else sel.numel()
        if n == 0:
            return None
        if n > s.rows:
            raise L.OmniError(f"logits of {n} rows from a batch of {T} tokens")
        nfrag = self.elem.code == 0 and n <= SKINNY
        final = dict(final_gain=self.final_norm) if isinstance(self.final_norm, float) else dict(final_w=self.final_norm)
        self._rows(**add, use_final=1, **final, sel=sel, h_out=s.hn, frag=int(nfrag), rows=n)
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
        b = Batch(B, B, self.input_ids, self.row_ids, self.positions, self.d.max_model_len, num_live=self.num_live)
        self.forward(b, logits=self.logits[:B], scratch=self._dec)
        if advance and self.d.vocab <= self.MAX_SAMPLED_VOCAB:
            self.sample_rows_in_place(B, self.num_live)

    # ------------------------------------------------------------------ roofline accounting
    def step_bytes(self, ctx_lens) -> dict:
        """Bytes a decode step must move: matrices of every layer run, the head, the cache read and written, the recurrent state read and written."""
        from .weights import decoder_weight_bytes
        es = torch.empty((), dtype=self.elem.torch).element_size()
        w = decoder_weight_bytes(self.d) * es // 2
        read = wrote = 0
        for c in ctx_lens:
            for i in range(self.d.num_layers):
                r, n = cache_traffic(self.d, i, int(c))
                read, wrote = read + r * es, wrote + n * es
        state = 2 * len(ctx_lens) * sum(state_bytes(self.d, i) for i in range(self.d.num_layers))
        return {"weights": w, "kv_read": read, "kv_write": wrote, "state": state, "total": w + read + wrote + state}
