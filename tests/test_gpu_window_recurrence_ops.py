"""Kernels of windowed grouped attention, the decaying recurrence, norms behind sums and the side input, each against the oracle's equation."""
import ctypes as C

import pytest
import torch

from ht_vllm_omni_amd import _lib as L
from ht_vllm_omni_amd import ops
from ht_vllm_omni_amd.decoder_mixers import attention_tiles, r32, recurrence_chunks, recurrence_segments, rotation_table
from ht_vllm_omni_amd.engine import frag_shuffle
from oracle import decoder_oracle as D
from tests.test_gpu_decoder_ops import ELEMS, RTOL, call, close, dev, frag_rows, gen, padc, run_struct, unfrag

pytestmark = pytest.mark.gpu
SAFE = {0: 8e-3, 1: 1e-5}


def pad_heads(t, heads, dim, dp):
    """[..., heads * dim] -> [..., heads * dp]"""
    return padc(t.reshape(*t.shape[:-1], heads, dim), dp).reshape(*t.shape[:-1], heads * dp)


def slabs_of(x, n, g):
    """n arrays whose sum is x, zeros where x is zero padding."""
    parts = torch.randn(n, *x.shape, generator=g) * (x != 0)
    parts[n - 1] = x - parts[:n - 1].sum(0)
    return parts


# ---------------------------------------------------------------- residual stream
@pytest.mark.parametrize("elem", [0, 1])
@pytest.mark.parametrize("width,T", [(40, 1), (136, 6), (1000, 70), (3000, 5)])
def test_norm_behind_the_sum(elem, width, T):
    g, wp = gen(width), r32(width)
    x, y = torch.randn(T, width, generator=g) * 3, torch.randn(T, width, generator=g)
    w = torch.randn(width, generator=g).to(ELEMS[elem])
    ref = D.post_norm(x.double(), y.double(), w.double(), 1.6, 1e-5)
    xo = torch.full((T, wp), 7.0, device="cuda")
    frag = int(elem == 0 and T <= 64)
    h = torch.zeros((T + 15) // 16 * 16, wp, dtype=ELEMS[elem], device="cuda")
    run_struct("omni_stream_rows_run", L.StreamRows(), x_in=dev(padc(x, wp)), y=dev(padc(slabs_of(y, 3, g), wp)), y_slabs=3, y_stride=T * wp, eps=1e-5, post=1, alpha=1.6, y_w=dev(padc(w, wp)),
               x_out=xo, h_out=h, frag=frag, rows=T, width=width, wp=wp, elem=elem)
    close(xo[:, :width], ref, 2e-6, "x")
    close((unfrag(h, T, wp) if frag else h[:T])[:, :width], ref, RTOL[elem], "h")
    assert not xo[:, width:].any(), "padding must stay zero"


@pytest.mark.parametrize("elem", [0, 1])
def test_weight_vectors_of_added_and_final_norms_and_scaled_embedding(elem):
    g, V, width = gen(5), 37, 72
    wp = r32(width)
    table = torch.randn(V, width, generator=g).to(ELEMS[elem])
    ids = torch.tensor([3, 36, 0, 7, 7], dtype=torch.int32)
    xo = torch.zeros(5, wp, device="cuda")
    run_struct("omni_stream_rows_run", L.StreamRows(), ids=dev(ids), table=dev(padc(table, wp)), vocab=V, table_scale=2.5, x_out=xo, rows=5, width=width, wp=wp, elem=elem)
    e = table[ids.long()].double() * 2.5
    close(xo[:, :width], e, 1e-7)
    y = torch.randn(5, width, generator=g)
    yw, fw = torch.randn(width, generator=g).to(ELEMS[elem]), torch.randn(width, generator=g).to(ELEMS[elem])
    sel = torch.tensor([4, 0, 2], dtype=torch.int32)
    out = torch.zeros(3, wp, dtype=ELEMS[elem], device="cuda")
    run_struct("omni_stream_rows_run", L.StreamRows(), x_in=xo, y=dev(padc(y, wp)), y_w=dev(padc(yw, wp)), eps=1e-6, use_final=1, final_w=dev(padc(fw, wp)), sel=dev(sel), h_out=out, rows=3, width=width,
               wp=wp, elem=elem)
    new = e + D.rms_norm(y.double(), yw.double(), 1e-6)
    close(out[:, :width], D.rms_norm(new, fw.double(), 1e-6)[sel.long()], RTOL[elem])


@pytest.mark.parametrize("elem,form", [(0, "sums"), (1, "sums"), (0, "rows")])
@pytest.mark.parametrize("heads,dim", [(1, 8), (3, 40), (16, 128), (20, 200)])
def test_gated_norm(elem, heads, dim, form):
    g, T, dp = gen(dim), 9, r32(dim)
    n = heads * dp
    o, z, w = torch.randn(T, heads * dim, generator=g), torch.randn(T, heads * dim, generator=g), torch.randn(heads * dim, generator=g).to(ELEMS[elem])
    ld = n + 64
    if form == "sums":
        full = torch.zeros(2, T, ld)
        full[:, :, 64:] = slabs_of(pad_heads(z, heads, dim, dp), 2, g)
        gate, slabs, s = dev(full), 2, torch.sigmoid(z.double())
    else:
        full = torch.zeros(T, ld, dtype=torch.bfloat16)
        full[:, 64:] = pad_heads(torch.sigmoid(z), heads, dim, dp).bfloat16()
        gate, slabs, s = dev(full), 0, torch.sigmoid(z).bfloat16().double()
    out = torch.zeros(16, n, dtype=ELEMS[elem], device="cuda")
    run_struct("omni_gated_norm_run", L.GatedNorm(), o=dev(pad_heads(o, heads, dim, dp)), w=dev(pad_heads(w, heads, dim, dp)), gate=gate.data_ptr() + 64 * gate.element_size(), slabs=slabs,
               slab_stride=T * ld, ld=ld, n=n, count=heads * dim, eps=1e-5, out=out, frag=int(elem == 0), T=T, elem=elem)
    got = unfrag(out, T, n) if elem == 0 else out[:T]
    close(got, pad_heads(D.rms_norm(o.double(), w.double(), 1e-5) * s, heads, dim, dp), RTOL[elem])


# ---------------------------------------------------------------- keys, values, rotation
@pytest.mark.parametrize("elem", [0, 1])
@pytest.mark.parametrize("heads,kv,dim,vdim,rot,own", [(1, 1, 8, 8, 2, True), (6, 2, 40, 24, 10, True), (6, 2, 40, 24, 40, False), (16, 4, 128, 128, 64, True), (20, 1, 72, 136, 0, True)])
def test_qkv_write(elem, heads, kv, dim, vdim, rot, own):
    """Norms over the whole projections, rotation at the tokens' positions, cache pages, gate; half a rotation that is no multiple of the vector width."""
    g, T, bs = gen(dim + rot), 9, 16
    dp, vp = r32(dim), r32(vdim)
    q, k, v, z = (torch.randn(T, h * n, generator=g) for h, n in ((heads, dim), (kv, dim), (kv, vdim), (heads, vdim)))
    parts = [pad_heads(q, heads, dim, dp)] + ([pad_heads(k, kv, dim, dp), pad_heads(v, kv, vdim, vp)] if own else []) + [pad_heads(z, heads, vdim, vp)]
    proj = torch.cat(parts, 1)
    ld = proj.shape[1]
    qw, kw = torch.randn(heads * dim, generator=g).to(ELEMS[elem]), torch.randn(kv * dim, generator=g).to(ELEMS[elem])
    row = torch.tensor([0, 1, 1, 1, 2, 2, 3, 3, 3], dtype=torch.int32)
    pos = torch.tensor([31, 15, 16, 17, 0, 1, 47, 48, 49], dtype=torch.int32)
    bt = torch.tensor([[5, 2, 9, 1], [3, 8, 4, 6], [7, 1, 1, 1], [9, 9, 9, 10]], dtype=torch.int32)
    live = torch.tensor([3], dtype=torch.int32)                                      # row 3 is padding
    kc = torch.full((11, kv, bs, dp), 5.0, dtype=ELEMS[elem], device="cuda")
    vc = torch.full((11, kv, bs, vp), 5.0, dtype=ELEMS[elem], device="cuda")
    qo, go = torch.zeros(T, heads * dp, dtype=ELEMS[elem], device="cuda"), torch.zeros(T, heads * vp, dtype=ELEMS[elem], device="cuda")
    run_struct("omni_qkv_write_run", L.QkvWrite(), proj=dev(slabs_of(proj, 2, g)), slabs=2, slab_stride=T * ld, ld=ld, heads=heads, kv_heads=kv, dim=dim, dp=dp, vp=vp, qw=dev(pad_heads(qw, heads, dim, dp)),
               kw=dev(pad_heads(kw, kv, dim, dp)), eps=1e-5, rot=dev(rotation_table(64, rot, 300.0)) if rot else None, rot_dims=rot, rot_rows=64, q=qo, kc=kc if own else None, vc=vc if own else None, gate=go,
               block_table=dev(bt), bt_stride=4, block_size=bs, row_of_tok=dev(row), positions=dev(pos), num_live=dev(live), T=T, elem=elem)

    def turned(x, h, w):
        n = D.rms_norm(x.double(), w.double(), 1e-5).reshape(T, h, dim)
        out = torch.zeros(64, h, dim, dtype=torch.double)
        res = []
        for t in range(T):                                                           # the oracle's rows are positions
            out.zero_()
            out[pos[t]] = n[t]
            res.append(D.rotate_half(out, rot, 300.0)[pos[t]] if rot else n[t])
        return torch.stack(res)
    close(qo.view(T, heads, dp)[:, :, :dim], turned(q, heads, qw), RTOL[elem], "q")
    assert not qo.view(T, heads, dp)[:, :, dim:].any()
    close(go.view(T, heads, vp)[:, :, :vdim], torch.sigmoid(z.double()).reshape(T, heads, vdim), RTOL[elem], "gate")
    wk, wv = torch.full((11, kv, bs, dp), 5.0, dtype=torch.double), torch.full((11, kv, bs, vp), 5.0, dtype=torch.double)
    if own:
        kk = turned(k, kv, kw)
        for t in range(6):
            wk[int(bt[row[t], pos[t] // bs]), :, int(pos[t]) % bs] = padc(kk[t], dp)
            wv[int(bt[row[t], pos[t] // bs]), :, int(pos[t]) % bs] = padc(v[t].double().reshape(kv, vdim), vp)
    close(kc, wk, RTOL[elem], "keys")
    close(vc, wv, RTOL[elem], "values")


# ---------------------------------------------------------------- epilogues
@pytest.mark.parametrize("M", [1, 17, 64, 65, 300])
@pytest.mark.parametrize("N,K", [(32, 64), (96, 32), (256, 320)])
def test_relu2_and_row_table_epilogues(M, N, K):
    g, V, off = gen(M + N), 23, 32
    x, w = (torch.randn(M, K, generator=g) / K ** 0.25).bfloat16(), (torch.randn(N, K, generator=g) / K ** 0.25).bfloat16()
    table = torch.randn(V, off + N, generator=g).bfloat16()
    ids = torch.randint(0, V, (M,), generator=g).to(torch.int32)
    z = x.double() @ w.double().T
    r2, side = torch.relu(z) ** 2, D.gelu_tanh(z) * table[ids.long()][:, off:].double()
    td, idd = dev(table), dev(ids)
    rt = L.RowTable(td.data_ptr() + 2 * off, idd.data_ptr(), V, off + N)
    lib = L.load_decoder()
    if M <= 64:
        xf, wf = frag_rows(x), frag_shuffle(dev(w))
        for frag in (0, 1):
            out = torch.zeros((M + 15) // 16 * 16, N, dtype=torch.bfloat16, device="cuda")
            call("omni_gemm_stream", xf, wf, out, M, N, K, L.STREAM_RELU2, 0, 0.0, 0.0, frag)
            close(unfrag(out, M, N) if frag else out[:M], r2, 8e-3, "relu2")
            call("omni_gemm_stream_rows", xf, wf, out, M, N, K, C.byref(rt), frag)
            close(unfrag(out, M, N) if frag else out[:M], side, 8e-3, "side")
    close(ops.gemm_tile(dev(x), frag_shuffle(dev(w)), act=L.TILE_ACT_RELU2, lib=lib), r2, 8e-3, "tile relu2")
    close(ops.gemm_tile(dev(x), frag_shuffle(dev(w)), act=L.TILE_ACT_GELU_MUL, mul=rt, lib=lib), side, 8e-3, "tile side")
    split = N // 2 // 16 * 16
    both = torch.cat([z[:, :split] * torch.sigmoid(z[:, :split]), torch.sigmoid(z[:, split:])], 1)
    close(ops.gemm_tile(dev(x), frag_shuffle(dev(w)), act=L.TILE_ACT_SILU_SIGMOID, act_cols=split, lib=lib), both, 8e-3, "tile silu | sigmoid")
    tf = dev(table.float())
    rt = L.RowTable(tf.data_ptr() + 4 * off, idd.data_ptr(), V, off + N)
    out = torch.zeros(M, N, device="cuda")
    call("omni_gemm_f32", dev(x.float()), K, 0, dev(w.float()), 0, out, N, 0, M, N, K, 1, L.ACT_RELU2, 0.0, 0.0)
    close(out, r2, 4e-6, "fp32 relu2")
    call("omni_gemm_f32_rows", dev(x.float()), K, dev(w.float()), out, N, M, N, K, C.byref(rt))
    close(out, side, 4e-6, "fp32 side")


# ---------------------------------------------------------------- attention
class Seqs:
    """Sequences of given lengths in a scrambled paged cache; the last `new[r]` tokens of each are the batch."""

    def __init__(self, lens, new, heads, kv, dim, vdim, elem, bs=16, seed=0, gated=True, sink=True):
        g = gen(seed)
        self.lens, self.new, self.heads, self.kv, self.dim, self.vdim, self.elem, self.bs = lens, new, heads, kv, dim, vdim, elem, bs
        E = ELEMS[elem]
        need = [(n + bs - 1) // bs for n in lens]
        ids = (torch.randperm(sum(need) + 3, generator=g) + 1).tolist()
        self.bt = torch.zeros(len(lens), max(need), dtype=torch.int32)
        self.k = [torch.randn(n, kv, dim, generator=g).to(E) for n in lens]
        self.v = [torch.randn(n, kv, vdim, generator=g).to(E) for n in lens]
        self.q = [(torch.randn(n, heads, dim, generator=g) * 0.5).to(E) for n in new]
        self.gate = torch.rand(sum(new), heads * vdim, generator=g).to(E) if gated else None
        self.sink = torch.randn(heads, generator=g) * 2 if sink else None
        self.blocks = len(ids) + 1
        for r in range(len(lens)):
            self.bt[r, :need[r]] = torch.tensor([ids.pop() for _ in range(need[r])])

    def caches(self):
        dp, vp, E = r32(self.dim), r32(self.vdim), ELEMS[self.elem]
        kc, vc = torch.full((self.blocks, self.kv, self.bs, dp), 9.0, dtype=E), torch.full((self.blocks, self.kv, self.bs, vp), 9.0, dtype=E)      # slots of no key hold large values
        for r, n in enumerate(self.lens):
            for j in range(n):
                b = int(self.bt[r, j // self.bs])
                kc[b, :, j % self.bs], vc[b, :, j % self.bs] = padc(self.k[r][j], dp), padc(self.v[r][j], vp)
        return kc, vc

    def reference(self, scale, window):
        out = []
        for r, (n, m) in enumerate(zip(self.lens, self.new)):
            q = torch.zeros(n, self.heads, self.dim, dtype=torch.double)
            q[n - m:] = self.q[r].double()
            out.append(D.window_attention(q, self.k[r].double(), self.v[r].double(), scale, window, None if self.sink is None else self.sink.double())[n - m:])
        out = torch.cat(out).reshape(-1, self.heads * self.vdim)
        return out if self.gate is None else out * self.gate.double()

    def run(self, scale, window, split=True, frag=0):
        order = sorted(range(len(self.lens)), key=lambda r: self.new[r] > 1)
        ones = sum(1 for n in self.new if n == 1)
        row = torch.cat([torch.full((self.new[r],), r) for r in order]).to(torch.int32)
        pos = torch.cat([torch.arange(self.lens[r] - self.new[r], self.lens[r]) for r in order]).to(torch.int32)
        base = [sum(self.new[:r]) for r in range(len(self.new))]
        perm = torch.cat([torch.arange(base[r], base[r] + self.new[r]) for r in order])
        dp, vp, H = r32(self.dim), r32(self.vdim), self.heads
        q = dev(padc(torch.cat([self.q[r] for r in order]), dp))
        gate = None if self.gate is None else dev(pad_heads(self.gate[perm], H, self.vdim, vp))
        T, starts, o = q.shape[0], [], ones
        seg = [self.new[r] for r in order[ones:]]
        for n in seg:
            starts.append(o)
            o += n
        lib = L.load_decoder()
        rows = lib.omni_window_attn_tile_rows(dp, vp)
        tiles = dev(torch.tensor(attention_tiles(starts, seg, H // self.kv, rows), dtype=torch.int32)) if seg else None
        out = torch.full(((T + 15) // 16 * 16, H * vp), float("nan"), dtype=ELEMS[self.elem], device="cuda")
        nb = lib.omni_window_attn_workspace_bytes(max(ones, 1), H, vp)
        kc, vc = self.caches()
        run_struct("omni_window_attn_run", L.WindowAttn(), q=q, kc=dev(kc), vc=dev(vc), gate=gate, sink=None if self.sink is None else dev(self.sink), out=out, frag=frag,
                   block_table=dev(self.bt), bt_stride=self.bt.shape[1], block_size=self.bs, row_of_tok=dev(row), positions=dev(pos), tiles=tiles, n_tiles=0 if tiles is None else len(tiles), tile_rows=rows,
                   T=T, n_decode=ones, heads=H, kv_heads=self.kv, dp=dp, vp=vp, scale=scale, window=window or 0, max_keys=max([self.lens[r] for r in order[:ones]] or [0]),
                   workspace=torch.full((nb // 4,), float("nan"), device="cuda") if split else None, workspace_bytes=nb if split else 0, elem=self.elem)
        got = (unfrag(out, T, H * vp) if frag else out[:T]).cpu().reshape(T, H, vp)
        assert not got[:, :, self.vdim:].any() or self.gate is None
        res = torch.empty(T, H * self.vdim, dtype=got.dtype)
        res[perm] = got[:, :, :self.vdim].reshape(T, -1)
        return res


SHAPES = [(1, 1, 8, 8), (6, 2, 40, 24), (4, 4, 64, 64), (9, 3, 80, 56), (16, 2, 128, 128), (20, 1, 72, 136), (8, 1, 256, 256)]


@pytest.mark.parametrize("elem", [0, 1])
@pytest.mark.parametrize("window", [None, 1, 5, 32, 100])
@pytest.mark.parametrize("heads,kv,dim,vdim", SHAPES + [(2, 1, 264, 288)])
def test_window_attention_over_mixed_batches(elem, window, heads, kv, dim, vdim):
    """Decoded tokens (one key, page borders, hundreds of keys) beside prompts and portions that start in the middle of a page or a tile."""
    s = Seqs([1, 16, 17, 300, 5, 33, 130, 97], [1, 1, 1, 1, 5, 33, 2, 40], heads, kv, dim, vdim, elem, seed=dim + heads)
    ref = s.reference(0.3, window)
    close(s.run(0.3, window), ref, SAFE[elem])
    if elem == 0:
        small = Seqs([1, 16, 300, 33], [1, 1, 1, 33], heads, kv, dim, vdim, elem, seed=dim, gated=False, sink=False)
        close(small.run(0.3, window, frag=1), small.reference(0.3, window), SAFE[elem], "fragment-major, no gate, no sink")


@pytest.mark.parametrize("elem,heads,kv,dim,vdim", [(0, 4, 2, 64, 32), (0, 10, 2, 80, 56), (0, 2, 2, 128, 136), (1, 2, 1, 40, 40)])
@pytest.mark.parametrize("window", [7, 16, 48])
def test_a_window_ends_exactly_where_it_ends(elem, heads, kv, dim, vdim, window):
    """One key stands out; it is seen by exactly the tokens whose window holds it -- in a decoded token, in a portion of three and in a prompt -- and the
    keys around it are ordinary.  A window one token off shows as the whole of that key's value."""
    n = 150
    for j in sorted({0, 15, 16, 31, 32, n - 1, n - 3, n - window - 2, n - window - 1, n - window, n - window + 1, n - window + 2}):
        if not 0 <= j < n:
            continue
        s = Seqs([n, n, n], [1, 3, n], heads, kv, dim, vdim, elem, seed=j)
        e = torch.zeros(dim)
        e[j % dim] = 6.0
        for r in range(3):
            s.k[r][:, :, j % dim] = 0
            s.k[r][j] = (s.k[r][j].float() * 0.1 + e).to(ELEMS[elem])
            s.q[r] = torch.zeros_like(s.q[r])
            s.q[r][..., j % dim] = 4.0
        ref = s.reference(1.0, window)
        close(s.run(1.0, window), ref, SAFE[elem], f"key {j}")
        seen = [j <= n - 1 and n - 1 - j < window] + [j <= i and i - j < window for i in (n - 3, n - 2, n - 1)]
        for a, t in zip(seen, range(4)):                                             # the planted key decides where it is seen
            v = s.v[0 if t == 0 else 1][j].double().repeat_interleave(heads // kv, 0).reshape(-1) * s.gate[t].double()
            assert a == bool((ref[t] - v).norm() < 0.05 * v.norm()), (j, t)


@pytest.mark.parametrize("elem", [0, 1])
def test_the_sink_takes_its_share(elem):
    """With a large number in the denominator the output shrinks towards zero, with a very small one it is plain attention, in every path."""
    s = Seqs([400, 20, 33], [1, 1, 33], 4, 2, 64, 64, elem, seed=3)
    outs = []
    for v in (-40.0, 0.0, 12.0):
        s.sink = torch.full((4,), v)
        got = s.run(0.2, None)
        close(got, s.reference(0.2, None), SAFE[elem], str(v))
        outs.append(float(got.float().norm()))
    assert outs[0] > 1.01 * outs[1] and outs[2] < 0.2 * outs[0]
    s.sink = None
    assert abs(float(s.run(0.2, None).float().norm()) / outs[0] - 1) < 1e-3


@pytest.mark.parametrize("window", [None, 700, 2049])
def test_splits_and_single_walk_agree(window):
    s = Seqs([2500, 40], [1, 1], 16, 2, 128, 128, 0, seed=4)
    ref = s.reference(0.15, window)
    for split in (True, False):
        close(s.run(0.15, window, split), ref, SAFE[0])


# ---------------------------------------------------------------- recurrence
def run_recurrence(lens, start, heads, dim, vdim, decay, form, seed=0, dead=(), tol=3e-6):
    """Sequences whose tokens [start, start + len) are the batch, the state of earlier ones in their slots (garbage where there are none)."""
    g = gen(seed)
    dp, vp, T = r32(dim), r32(vdim), sum(lens)
    total = [s + n for s, n in zip(start, lens)]
    raw = form == "sums"
    q, k, v = [], [], []
    for n in total:
        for lst, w in ((q, dim), (k, dim), (v, vdim)):
            z = torch.randn(n, heads, w, generator=g)
            lst.append(z if raw else torch.nn.functional.silu(z).bfloat16())
    act = (lambda z: torch.nn.functional.silu(z.double())) if raw else (lambda z: z.double())
    slot = (torch.randperm(len(lens), generator=g) + 1).to(torch.int32)
    state = torch.full((len(lens) + 2, heads, dp, vp), 77.0)
    ref, want = [], state.double().clone()
    for r, (s, n) in enumerate(zip(start, lens)):
        a, b, c = act(q[r]), act(k[r]), act(v[r])
        full = D.decay_recurrence(a, b, c, decay)
        for h in range(heads):
            S = torch.zeros(dim, vdim, dtype=torch.double)
            for t in range(total[r]):
                if t == s and s:
                    state[slot[r], h] = 0
                    state[slot[r], h, :dim, :vdim] = S.float()
                    want[slot[r], h] = state[slot[r], h].double()
                S = decay[h] * S + b[t, h][:, None] * c[t, h][None]
            if r not in dead:
                want[slot[r], h] = 0
                want[slot[r], h, :dim, :vdim] = S
        ref.append(full[s:])
    cols = [torch.cat([pad_heads(x[r][start[r]:].reshape(lens[r], -1), heads, w, p) for r in range(len(lens))]) for x, w, p in ((q, dim, dp), (k, dim, dp), (v, vdim, vp))]
    proj = torch.cat(cols + [torch.zeros(T, heads * vp, dtype=cols[0].dtype)], 1)
    ld = proj.shape[1]
    ones = 0
    while ones < len(lens) and lens[ones] == 1:
        ones += 1
    starts, o = [], ones
    for n in lens[ones:]:
        starts.append(o)
        o += n
    row = torch.cat([torch.full((n,), r) for r, n in enumerate(lens)]).to(torch.int32)
    pos = torch.cat([torch.arange(s, s + n) for s, n in zip(start, lens)]).to(torch.int32)
    a = dict(proj=dev(slabs_of(proj, 3, g)) if raw else dev(proj), slabs=3 if raw else 0, slab_stride=T * ld, ld=ld, heads=heads, dp=dp, vp=vp, decay=dev(torch.tensor(decay)),
             log2_decay=dev(torch.tensor(decay, dtype=torch.double).log2().float()), state_slot=dev(slot), row_of_tok=dev(row), positions=dev(pos), n_decode=ones)
    if form == "chunks" and starts:
        ch, sg = recurrence_chunks(starts, lens[ones:]), recurrence_segments(starts, lens[ones:])
        a.update(chunks=dev(torch.tensor(ch, dtype=torch.int32)), n_chunks=len(ch), segs=dev(torch.tensor(sg, dtype=torch.int32)), n_segs=len(sg),
                 chunk_states=torch.full((len(ch) * heads * dp * vp,), float("nan"), device="cuda"))
    elif starts:
        a.update(runs=dev(torch.tensor(list(zip(starts, lens[ones:])), dtype=torch.int32)), n_runs=len(starts))
    if dead:
        a["num_live"] = dev(torch.tensor([min(dead)], dtype=torch.int32))
    std, out = dev(state), torch.zeros(T, heads * vp, device="cuda")
    run_struct("omni_decay_rec_run", L.DecayRec(), state=std, out=out, **a)
    got = out.view(T, heads, vp)[:, :, :vdim].cpu()
    alive = torch.cat([torch.full((n,), r not in dead) for r, n in enumerate(lens)])
    close(got[alive], torch.cat(ref)[alive], tol, "out")
    close(std, want, tol, "state")
    assert not out.view(T, heads, vp)[:, :, vdim:].any()


DECAYS = [0.6, 0.9, 0.999, 1.0, 0.05]


@pytest.mark.parametrize("form", ["sums", "rows", "chunks"])
@pytest.mark.parametrize("heads,dim,vdim", [(1, 8, 8), (3, 24, 40), (2, 64, 64), (2, 128, 128), (2, 136, 200), (1, 256, 256)])
def test_recurrence_over_mixed_batches(form, heads, dim, vdim):
    """Decoded tokens and portions, new sequences over slots that hold something else, carried state, chunks that are whole, partial and one token."""
    run_recurrence([1, 1, 5, 128, 129, 300, 2], [0, 7, 3, 0, 60, 0, 130], heads, dim, vdim, DECAYS[:heads] if heads > 1 else [0.97], form, seed=dim)


@pytest.mark.parametrize("form", ["sums", "rows"])
def test_recurrence_with_heads_wider_than_a_chunk_takes(form):
    run_recurrence([1, 40], [3, 2], 1, 500, 288, [0.9], form)


@pytest.mark.parametrize("form", ["sums", "chunks"])
def test_recurrence_remembers_and_forgets(form):
    """Decays from keeping everything to forgetting at once, over 520 tokens: nothing over- or underflows into the result."""
    run_recurrence([520], [0], 5, 32, 32, DECAYS, form, seed=9, tol=1e-5)          # (hundreds of fp32 sums without decay)
    run_recurrence([400], [40], 3, 32, 32, [1e-3, 1e-30, 1.0], form, seed=10, tol=1e-5)


def test_rows_past_the_live_count_keep_their_state():
    run_recurrence([1, 1, 1, 1], [4, 0, 9, 2], 2, 40, 24, [0.9, 0.7], "sums", dead=(2, 3))


def test_argument_errors_come_back_as_errors():
    lib = L.load_decoder()
    for fn, s in (("omni_qkv_write_run", L.QkvWrite()), ("omni_gated_norm_run", L.GatedNorm()), ("omni_window_attn_run", L.WindowAttn()), ("omni_decay_rec_run", L.DecayRec())):
        assert getattr(lib, fn)(C.byref(s), None) == -1
    x = torch.zeros(64, 64, device="cuda")
    z = torch.zeros(8, dtype=torch.int32, device="cuda")
    p = x.data_ptr()
    a = L.WindowAttn(q=p, kc=p, vc=p, out=p, block_table=z.data_ptr(), row_of_tok=z.data_ptr(), positions=z.data_ptr(), bt_stride=1, block_size=16, heads=3, kv_heads=2, dp=32, vp=32, T=1, n_decode=1)
    assert lib.omni_window_attn_run(C.byref(a), None) == -1 and b"heads" in lib.omni_last_error()
    b = L.StreamRows(x_in=p, x_out=p + 4096, rows=1, width=32, wp=32, elem=1, post=1)
    assert lib.omni_stream_rows_run(C.byref(b), None) == -1 and b"behind the sum" in lib.omni_last_error()
    assert lib.omni_gemm_stream_rows(p, p, p, 1, 32, 32, None, 0, None) == -1
    assert lib.omni_gemm_f32_rows(p, 32, p, p, 32, 1, 32, 32, None, None) == -1
