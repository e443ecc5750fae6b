"""Kernels of the decoder-only language models, each against the oracle's equation of the same mechanism."""
import ctypes as C

import pytest
import torch

from ht_vllm_omni_amd import _lib as L
from ht_vllm_omni_amd import ops
from ht_vllm_omni_amd.decoder_engine import attention_tiles, r32
from ht_vllm_omni_amd.engine import frag_shuffle, frag_unshuffle
from oracle import decoder_oracle as D

pytestmark = pytest.mark.gpu
ELEMS = {0: torch.bfloat16, 1: torch.float32}
RTOL = {0: 8e-3, 1: 4e-6}


def gen(seed):
    return torch.Generator().manual_seed(seed)


def close(got, ref, tol, what=""):
    g, r = got.double().cpu(), ref.double().cpu()
    assert g.shape == r.shape, (what, g.shape, r.shape)
    err = (g - r).abs().max() / r.abs().max().clamp_min(1e-6)
    assert torch.isfinite(g).all() and float(err) <= tol, f"{what}: {float(err):.3g} > {tol}"


def dev(t, dt=None):
    return t.to(device="cuda", dtype=dt or t.dtype).contiguous()


def call(fn, *a):
    """Tensors are passed as they are: the argument list keeps them alive until the kernel has run."""
    lib = L.load_decoder()
    L.check(getattr(lib, fn)(*[L.ptr(v) if isinstance(v, torch.Tensor) else v for v in a], L.current_stream()), fn, lib)
    torch.cuda.synchronize()


def run_struct(fn, s, **kw):
    for k, v in kw.items():
        setattr(s, k, L.ptr(v) if isinstance(v, torch.Tensor) else v)
    call(fn, C.byref(s))


def padc(t, n):
    out = torch.zeros(*t.shape[:-1], n, dtype=t.dtype)
    out[..., :t.shape[-1]] = t
    return out


def unfrag(h, rows, width):
    return frag_unshuffle(h.view(-1, width))[:rows]


# ---------------------------------------------------------------- residual stream, shift, norms
@pytest.mark.parametrize("elem", [0, 1])
@pytest.mark.parametrize("width,segs", [(40, [1]), (136, [3, 1, 2]), (1000, [5, 17]), (2048, [1, 1, 1]), (3000, [2, 9]), (264, [1100, 1, 2, 33])])
def test_stream_rows_norm_add_and_shift(elem, width, segs):
    """x += g y / rms(y), then the shift: a batch's first token of a sequence takes the state (or zeros at position 0), the others their
    neighbour's NEW row."""
    g, wp, T = gen(width), r32(width), sum(segs)
    x, y = torch.randn(T, width, generator=g) * 3, torch.randn(T, width, generator=g)
    mu = torch.rand(width, generator=g).to(ELEMS[elem])
    state = torch.randn(len(segs) + 2, width, generator=g)
    slot = torch.randperm(len(segs), generator=g).to(torch.int32) + 1
    row = torch.cat([torch.full((n,), r) for r, n in enumerate(segs)]).to(torch.int32)
    start = [0 if r % 2 == 0 else 11 for r in range(len(segs))]                       # even rows begin their sequence in this batch
    pos = torch.cat([torch.arange(s, s + n) for s, n in zip(start, segs)]).to(torch.int32)
    new = x.double() + D.scalar_rms_norm(y.double(), torch.tensor(0.7).double(), 1e-5)
    ref, o = [], 0
    for r, n in enumerate(segs):
        before = new.new_zeros(1, width) if start[r] == 0 else state[slot[r]].double()[None]
        ref.append(D.token_shift(torch.cat([before, new[o:o + n]]), mu.double())[1:])
        o += n
    xo = torch.full((T, wp), 7.0, device="cuda")
    frag = int(elem == 0 and T <= 64)
    h = torch.zeros((T + 15) // 16 * 16, wp, dtype=ELEMS[elem], device="cuda")
    parts = torch.randn(3, T, width, generator=g)                                    # y arrives as three partial sums
    parts[2] = y - parts[0] - parts[1]
    run_struct("omni_stream_rows_run", L.StreamRows(), x_in=dev(padc(x, wp)), y=dev(padc(parts, wp)), y_slabs=3, y_stride=T * wp, gain=0.7, eps=1e-5, mu=dev(padc(mu, wp)), state=dev(padc(state, wp)),
               state_slot=dev(slot), row_of_tok=dev(row), positions=dev(pos), x_out=xo, h_out=h, frag=frag, rows=T, width=width, wp=wp, elem=elem)
    close(xo[:, :width], new, 1e-6, "x")
    hh = unfrag(h, T, wp) if frag else h[:T]
    close(hh[:, :width], torch.cat(ref), RTOL[elem], "h")
    assert not xo[:, width:].any() and not hh[:, width:].any(), "padding must stay zero"


@pytest.mark.parametrize("elem", [0, 1])
def test_stream_rows_embedding_and_final_norm(elem):
    g, V, width = gen(5), 37, 72
    wp = r32(width)
    table = torch.randn(V, width, generator=g).to(ELEMS[elem])
    ids = torch.tensor([3, 36, 0, 7, 7], dtype=torch.int32)
    mu = torch.rand(width, generator=g).to(ELEMS[elem])
    xo, h = torch.zeros(5, wp, device="cuda"), torch.zeros(5, wp, dtype=ELEMS[elem], device="cuda")
    z = torch.zeros(5, dtype=torch.int32, device="cuda")
    run_struct("omni_stream_rows_run", L.StreamRows(), ids=dev(ids), table=dev(padc(table, wp)), vocab=V, mu=dev(padc(mu, wp)), state=torch.zeros(2, wp, device="cuda"), state_slot=z,
               row_of_tok=z, positions=torch.arange(5, dtype=torch.int32, device="cuda"), x_out=xo, h_out=h, rows=5, width=width, wp=wp, elem=elem)
    e = table[ids.long()].double()
    close(xo[:, :width], e, 1e-7)
    close(h[:, :width], D.token_shift(e, mu.double()), RTOL[elem])
    y = torch.randn(5, width, generator=g)
    sel = torch.tensor([4, 0, 2], dtype=torch.int32)
    out = torch.zeros(3, wp, dtype=ELEMS[elem], device="cuda")
    run_struct("omni_stream_rows_run", L.StreamRows(), x_in=xo, y=dev(padc(y, wp)), gain=1.3, eps=1e-6, use_final=1, final_gain=0.9, sel=dev(sel), h_out=out, rows=3, width=width, wp=wp, elem=elem)
    new = e + D.scalar_rms_norm(y.double(), torch.tensor(1.3).double(), 1e-6)
    close(out[:, :width], D.scalar_rms_norm(new, torch.tensor(0.9).double(), 1e-6)[sel.long()], RTOL[elem])


@pytest.mark.parametrize("elem", [0, 1])
@pytest.mark.parametrize("q_rank,kv_rank,heads,gated", [(8, 8, 1, True), (48, 56, 3, False), (1500, 500, 33, True), (160, 264, 20, False)])
def test_latent_write(elem, q_rank, kv_rank, heads, gated):
    g, T, bs, width = gen(q_rank), 9, 16, 72
    qp, rp, wp = r32(q_rank), r32(kv_rank), r32(width)
    ld = qp + rp + (r32(heads) if gated else 0)
    proj = torch.zeros(T, ld)
    proj[:, :q_rank], proj[:, qp:qp + kv_rank] = torch.randn(T, q_rank, generator=g), torch.randn(T, kv_rank, generator=g) * 2
    if gated:
        proj[:, qp + rp:qp + rp + heads] = torch.randn(T, heads, generator=g)
    qw, kw = torch.randn(q_rank, generator=g).to(ELEMS[elem]), torch.randn(kv_rank, generator=g).to(ELEMS[elem])
    row = torch.tensor([0, 1, 1, 1, 2, 2, 3, 3, 3], dtype=torch.int32)
    pos = torch.tensor([31, 15, 16, 17, 0, 1, 47, 48, 49], dtype=torch.int32)
    bt = torch.tensor([[5, 2, 9, 1], [3, 8, 4, 6], [7, 1, 1, 1], [9, 9, 9, 10]], dtype=torch.int32)
    slot, live = torch.tensor([4, 2, 1, 3], dtype=torch.int32), torch.tensor([3], dtype=torch.int32)      # row 3 is padding
    x = torch.randn(T, width, generator=g)
    cq = torch.zeros((T + 15) // 16 * 16, qp, dtype=ELEMS[elem], device="cuda")
    cache = torch.full((11, bs, rp), 5.0, dtype=ELEMS[elem], device="cuda")
    gate, state = torch.zeros(T, heads, device="cuda"), torch.full((5, wp), 5.0, device="cuda")
    parts = torch.randn(2, T, ld, generator=g) * (proj != 0)                         # two partial sums
    parts[1] = proj - parts[0]
    run_struct("omni_latent_write_run", L.LatentWrite(), proj=dev(parts), slabs=2, slab_stride=T * ld, ld=ld, q_rank=q_rank, qp=qp, kv_rank=kv_rank, rp=rp, heads=heads, qw=dev(padc(qw, qp)), kw=dev(padc(kw, rp)),
               eps=1e-5, cq=cq, frag=int(elem == 0), cache=cache, gate=gate if gated else None, block_table=dev(bt), bt_stride=4, block_size=bs, row_of_tok=dev(row), positions=dev(pos),
               num_live=dev(live), x=dev(padc(x, wp)), wp=wp, state=state, state_slot=dev(slot), T=T, elem=elem)
    got = unfrag(cq, T, qp) if elem == 0 else cq[:T]
    close(got[:, :q_rank], D.rms_norm(proj[:, :q_rank].double(), qw.double(), 1e-5), RTOL[elem], "cq")
    c = D.rms_norm(proj[:, qp:qp + kv_rank].double(), kw.double(), 1e-5)
    want, written = torch.full((11, bs, rp), 5.0, dtype=torch.double), 0
    for t in range(T):
        if int(row[t]) < 3:
            want[int(bt[row[t], pos[t] // bs]), int(pos[t]) % bs] = padc(c[t], rp)
            written += 1
    assert written == 6
    close(cache, want, RTOL[elem], "cache")
    if gated:
        close(gate, torch.sigmoid(proj[:, qp + rp:qp + rp + heads].double()), 1e-6, "gate")
    ws = torch.full((5, wp), 5.0)
    for r, t in ((0, 0), (1, 3), (2, 5)):
        ws[slot[r]] = padc(x[t], wp)
    assert torch.equal(state.cpu(), ws), "state: each live sequence's last token, nothing else"


# ---------------------------------------------------------------- products
@pytest.mark.parametrize("T", [1, 7, 16, 33, 64, 200])
@pytest.mark.parametrize("heads,n,k", [(1, 32, 32), (3, 64, 32), (5, 48, 96), (16, 512, 128), (16, 128, 512), (2, 16, 288)])
def test_head_gemm(T, heads, n, k):
    g = gen(T + n)
    x, w = torch.randn(T, heads, k, generator=g).bfloat16(), torch.randn(heads, n, k, generator=g).bfloat16()
    ref = torch.stack([x[:, h].float() @ w[h].float().T for h in range(heads)], 1)
    frag = int(T <= 64 and heads * n % 32 == 0)
    out = torch.zeros((T + 15) // 16 * 16, heads * n, dtype=torch.bfloat16, device="cuda")
    call("omni_head_gemm", dev(x), frag_shuffle(dev(w)), out, T, heads, n, k, frag)
    torch.cuda.synchronize()
    got = unfrag(out, T, heads * n) if frag else out[:T]
    close(got.view(T, heads, n), ref, 8e-3)


@pytest.mark.parametrize("T,heads,n,k", [(70, 3, 64, 32), (512, 16, 512, 128), (600, 5, 48, 96), (130, 16, 128, 512)])
def test_tile_gemm_column_groups(T, heads, n, k):
    """One product per head of a [tokens, heads * k] array: the groups' rows are the same, their columns differ."""
    g = gen(T)
    x, w = torch.randn(T, heads, k, generator=g).bfloat16(), torch.randn(heads, n, k, generator=g).bfloat16()
    ref = torch.stack([x[:, h].float() @ w[h].float().T for h in range(heads)], 1)
    for want in "bf":
        out = ops.gemm_tile(dev(x).view(T, heads * k), frag_shuffle(dev(w)), groups=heads, group_cols=True, want=want, lib=L.load_decoder())
        close(out.view(T, heads, n), ref, 8e-3 if want == "b" else 2e-5)
    with pytest.raises(L.OmniError, match="group columns"):                  # rows of the output too short for the last head
        ops.gemm_tile(dev(x).view(T, heads * k), frag_shuffle(dev(w)), groups=heads, group_cols=True, lib=L.load_decoder(),
                      out=torch.zeros(T, heads * n - 8, dtype=torch.bfloat16, device="cuda"))


@pytest.mark.parametrize("M,N,K", [(1, 32, 32), (5, 77, 40), (130, 203, 136), (64, 512, 96)])
def test_gemm_f32_is_true_32_bit(M, N, K):
    g = gen(M)
    x, w = torch.randn(M, K, generator=g), torch.randn(N, K, generator=g)
    out = torch.zeros(M, N, device="cuda")
    call("omni_gemm_f32", dev(x), K, 0, dev(w), 0, out, N, 0, M, N, K, 1, 0, 0.0, 0.0)
    close(out, x.double() @ w.double().T, 2e-6)
    pq = torch.tensor([0.3, -0.8], dtype=torch.double)
    ap, an = torch.nn.functional.softplus(pq).tolist()
    call("omni_gemm_f32", dev(x), K, 0, dev(w), 0, out, N, 0, M, N, K, 1, 1, ap, 0.5 + an)
    close(out, D.xielu(x.double() @ w.double().T, pq), 2e-6)


def frag_rows(x):
    """Row-major [M, K] bf16 -> fragment-major in whole 16-row tiles; the rows past M hold values nothing may read."""
    M, K = x.shape
    full = torch.full(((M + 15) // 16 * 16, K), float("nan"), dtype=x.dtype)
    full[:M] = x
    return frag_shuffle(dev(full))


@pytest.mark.parametrize("M", [1, 15, 16, 17, 33, 48, 64])
@pytest.mark.parametrize("N,K", [(16, 32), (96, 64), (224, 288), (2080, 2048), (2048, 1536), (512, 4640), (9216, 256)])
def test_gemm_stream(M, N, K):
    """Every row-tile count, K that divides into nothing, partial sums over K, one sum, bf16 in both layouts, the activation."""
    g = gen(M * N)
    x, w = torch.randn(M, K, generator=g).bfloat16(), torch.randn(N, K, generator=g).bfloat16()
    ref = x.double() @ w.double().T
    xf, wf = frag_rows(x), frag_shuffle(dev(w))
    S = L.load_decoder().omni_gemm_stream_splits(M, N, K)
    assert 1 <= S <= L.STREAM_MAX_SPLITS
    out = torch.full((S, M, N), float("nan"), device="cuda")
    call("omni_gemm_stream", xf, wf, out, M, N, K, L.STREAM_F32, 0, 0.0, 0.0, 0)
    close(out.double().sum(0), ref, 2e-5)
    call("omni_gemm_stream", xf, wf, out, M, N, K, L.STREAM_F32, 1, 0.0, 0.0, 0)
    close(out[0], ref, 2e-5)
    b = torch.zeros((M + 15) // 16 * 16, N, dtype=torch.bfloat16, device="cuda")
    call("omni_gemm_stream", xf, wf, b, M, N, K, L.STREAM_BF16, 0, 0.0, 0.0, 0)
    close(b[:M], ref, 8e-3)
    if N % 32 == 0:
        call("omni_gemm_stream", xf, wf, b, M, N, K, L.STREAM_BF16, 0, 0.0, 0.0, 1)
        close(unfrag(b, M, N), ref, 8e-3)


@pytest.mark.parametrize("M", [1, 17, 64, 65, 300])
def test_xielu_epilogues(M):
    """The activation inside both GEMMs, over values far into either branch and around zero."""
    g, N, K = gen(M), 96, 64
    x, w = (torch.randn(M, K, generator=g) * 2).bfloat16(), torch.randn(N, K, generator=g).bfloat16()
    x[0], w[:5] = 1e-3, 1.0
    pq = torch.tensor([0.9, 0.2], dtype=torch.double)
    ap, an = torch.nn.functional.softplus(pq).tolist()
    ref = D.xielu(x.double() @ w.double().T, pq)
    if M <= 64:
        out = torch.zeros(M, N, dtype=torch.bfloat16, device="cuda")
        call("omni_gemm_stream", frag_rows(x), frag_shuffle(dev(w)), out, M, N, K, L.STREAM_XIELU, 0, ap, 0.5 + an, 0)
    else:
        out = ops.gemm_tile(dev(x), frag_shuffle(dev(w)), act=L.TILE_ACT_XIELU, act_params=(ap, 0.5 + an), lib=L.load_decoder())
    err = (out.double().cpu() - ref).abs() / ref.abs().clamp_min(2e-2)
    assert float(err.max()) <= 8e-3, float(err.max())


# ---------------------------------------------------------------- attention
class Seqs:
    """Sequences of given lengths in a scrambled paged cache; the last `new[r]` tokens of each are the batch."""

    def __init__(self, lens, new, heads, rp, elem, bs=16, seed=0):
        g = gen(seed)
        self.lens, self.new, self.heads, self.rp, self.elem, self.bs = lens, new, heads, rp, elem, bs
        need = [(n + bs - 1) // bs for n in lens]
        ids = (torch.randperm(sum(need) + 3, generator=g) + 1).tolist()
        stride = max(need)
        self.bt = torch.zeros(len(lens), stride, dtype=torch.int32)
        self.c = [torch.randn(n, rp, generator=g).to(ELEMS[elem]) for n in lens]
        self.q = [(torch.randn(k, heads, rp, generator=g) * 0.3).to(ELEMS[elem]) for k in new]
        self.cache = torch.full((len(ids) + 1, bs, rp), 9.0, dtype=ELEMS[elem])          # slots that belong to no key hold large values
        for r, n in enumerate(lens):
            blocks = [ids.pop() for _ in range(need[r])]
            self.bt[r, :len(blocks)] = torch.tensor(blocks)
            for j in range(n):
                self.cache[blocks[j // bs], j % bs] = self.c[r][j]
        self.gate = torch.rand(sum(new), heads, generator=g)

    def reference(self, scale):
        out = []
        for c, q, n, k in zip(self.c, self.q, self.lens, self.new):
            qq = torch.zeros(n, self.heads, self.rp, dtype=torch.double)
            qq[n - k:] = q.double()
            kv = c.double()[:, None].expand(n, self.heads, self.rp)
            out.append(D.causal_softmax_attention(qq, kv, kv, scale)[n - k:])
        return torch.cat(out) * self.gate[:, :, None]

    def run(self, scale, split=True):
        """Single-token sequences first, as the engine orders them."""
        order = sorted(range(len(self.lens)), key=lambda r: self.new[r] > 1)
        ones = sum(1 for n in self.new if n == 1)
        row = torch.cat([torch.full((self.new[r],), r) for r in order]).to(torch.int32)
        pos = torch.cat([torch.arange(self.lens[r] - self.new[r], self.lens[r]) for r in order]).to(torch.int32)
        base = [sum(self.new[:r]) for r in range(len(self.new))]
        perm = torch.cat([torch.arange(base[r], base[r] + self.new[r]) for r in order])
        q = dev(torch.cat([self.q[r] for r in order]))
        T = q.shape[0]
        starts, o = [], ones
        seg = [self.new[r] for r in order[ones:]]
        for n in seg:
            starts.append(o)
            o += n
        tile_rows = L.load_decoder().omni_latent_attn_tile_rows(self.rp)
        tiles = dev(torch.tensor(attention_tiles(starts, seg, self.heads, tile_rows), dtype=torch.int32)) if seg else None
        out = torch.full_like(q, float("nan"))
        nb = L.load_decoder().omni_latent_attn_workspace_bytes(max(ones, 1), self.heads, self.rp)
        ws = torch.full((nb // 4,), float("nan"), device="cuda") if split else None
        keep = [dev(self.cache), dev(self.gate[perm]), dev(self.bt), dev(row), dev(pos)]
        run_struct("omni_latent_attn_run", L.LatentAttn(), q=q, cache=keep[0], gate=keep[1], out=out, block_table=keep[2], bt_stride=self.bt.shape[1], block_size=self.bs,
                   row_of_tok=keep[3], positions=keep[4], tiles=tiles, n_tiles=0 if tiles is None else len(tiles), tile_rows=tile_rows, T=T, n_decode=ones, heads=self.heads, rp=self.rp, scale=scale,
                   max_keys=max([self.lens[r] for r in order[:ones]] or [0]), workspace=ws, workspace_bytes=nb if split else 0, elem=self.elem)
        torch.cuda.synchronize()
        res = torch.empty_like(out, device="cpu")
        res[perm] = out.cpu()
        return res


ATTN_TOL = {0: 8e-3, 1: 1e-5}


@pytest.mark.parametrize("elem,rp", [(0, 32), (0, 64), (0, 96), (0, 160), (0, 224), (0, 256), (0, 320), (0, 384), (0, 448), (0, 512), (0, 544), (1, 32), (1, 96), (1, 288)])
@pytest.mark.parametrize("heads", [1, 3, 16, 20])
def test_latent_attention_over_mixed_batches(elem, rp, heads):
    """Decoded tokens (one key, page borders, hundreds of keys) beside prompts and portions that start in the middle of a page or a tile."""
    s = Seqs([1, 16, 17, 300, 5, 33, 130, 97], [1, 1, 1, 1, 5, 33, 2, 40], heads, rp, elem, seed=rp + heads)
    close(s.run(0.4), s.reference(0.4), ATTN_TOL[elem])


@pytest.mark.parametrize("elem,rp,heads", [(0, 64, 4), (0, 512, 16), (1, 64, 2)])
def test_every_key_counts_exactly_once(elem, rp, heads):
    """Queries that single one key out: at every page border, tile border, the first token, the newest, and -- planted just past the end --
    none of a key that is not visible."""
    n = 261
    for j in [0, 1, 15, 16, 31, 32, 63, 64, 127, 128, 129, 255, 256, 259, 260]:
        s = Seqs([n, n, 40], [1, 3, 1], heads, rp, elem, seed=j)
        for r in (0, 1):
            d = torch.zeros(rp)
            d[j % rp] = 6.0
            s.c[r][j] = (s.c[r][j].float() + d).to(ELEMS[elem])
            s.cache[int(s.bt[r, j // 16]), j % 16] = s.c[r][j]
            s.q[r] = s.q[r] * 0
            s.q[r][..., j % rp] = 4.0
        ref = s.reference(1.0)
        close(s.run(1.0), ref, ATTN_TOL[elem], f"key {j}")
        # the marked key dominates for every row that sees it: a row that missed it (or saw one too many) would be far off
        seen = torch.tensor([True] + [n - 3 + i >= j for i in range(3)])
        assert (ref[:4][seen].norm(dim=-1) > 0).all()


def test_splits_and_single_walk_agree():
    s = Seqs([2500], [1], 16, 512, 0, seed=4)
    ref = s.reference(0.3)
    for split in (True, False):
        close(s.run(0.3, split), ref, ATTN_TOL[0])


def test_argument_errors_come_back_as_errors():
    lib = L.load_decoder()
    assert lib.omni_latent_attn_run(C.byref(L.LatentAttn()), None) == -1
    assert lib.omni_stream_rows_run(C.byref(L.StreamRows()), None) == -1
    assert lib.omni_latent_write_run(C.byref(L.LatentWrite()), None) == -1
    x = torch.zeros(4, 32, device="cuda")
    s = L.StreamRows(x_in=x.data_ptr(), x_out=x.data_ptr(), rows=4, width=32, wp=32, elem=1)
    assert lib.omni_stream_rows_run(C.byref(s), None) == -1 and b"x_in" in lib.omni_last_error()
    assert lib.omni_head_gemm(x.data_ptr(), x.data_ptr(), x.data_ptr(), 1, 1, 8, 32, 0, None) == -1
