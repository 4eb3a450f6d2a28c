"""Rudazen on the GPU against the plain implementation: every mechanism alone through its
kernel, then whole models (three small configurations, in 32-bit and in bfloat16) layer by
layer, whole, decoded token by token, in portions down to two tokens, in mixed batches with
pages and state slots that are given back and used again, from a captured graph, generated
greedily through the scheduler, through the trace replay program, and configurations drawn at
random. bfloat16 is compared with the plain implementation on the bfloat16-rounded weights."""
import json
import math
import os
import subprocess
import sys

import pytest
import torch

import plain_rudazen as plain
import rudazen_cases
import util

pytestmark = pytest.mark.gpu
DEV = "cuda"
STD = 0.25
D = torch.float64
KERNELS = [(torch.float32, False), (torch.bfloat16, False), (torch.bfloat16, True)]


@pytest.fixture(scope="module")
def ops():
    from ninfer_amd.kernels import load_ops
    return load_ops()


@pytest.fixture
def plain_kernel(request, ops):
    ops.force_generic = bool(getattr(request, "param", False))
    yield ops.force_generic
    ops.force_generic = False


def rel_err(got, want):
    got, want = got.double().cpu(), want.double().cpu()
    return ((got - want).norm() / want.norm().clamp_min(1e-30)).item()


def _cut(n, sizes, tail):
    """n rows as portions of the given sizes in turn, the last `tail` one by one."""
    out, i, j = [], 0, 0
    while i < n - tail:
        s = min(sizes[j % len(sizes)], n - tail - i)
        out.append(s)
        i += s
        j += 1
    return out + [1] * tail


def _steps(ops, dtype, cuts, slots):
    """StepContexts for requests that go on from step to step; cuts[r]: request r's portions.
    Requests that bring one row come first in a step, as the engine orders them."""
    done = [0] * len(cuts)
    for i in range(max(len(c) for c in cuts)):
        who = [r for r, c in enumerate(cuts) if i < len(c)]
        who.sort(key=lambda r: cuts[r][i] != 1)
        ctx = util.make_context(ops, dtype, [(done[r], cuts[r][i]) for r in who])
        ctx.seq_slots = torch.tensor([slots[r] for r in who], dtype=torch.int32, device=DEV)
        ctx.single_rows = sum(1 for r in who if cuts[r][i] == 1)
        yield ctx, who, [done[r] for r in who], [cuts[r][i] for r in who]
        for r in who:
            done[r] += cuts[r][i]


# ---- mechanisms alone ------------------------------------------------------------------------

@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("width", [70, 256, 1100, 5000])
def test_norm_behind_the_sum(ops, dtype, width):
    """x <- norm(alpha x + y) in 32-bit and in the activation dtype, y a row, the weighted sum of
    an expert's rows, or half the sum of two rows that are normed by themselves."""
    from ninfer_amd.parts import NormedSum
    g = torch.Generator().manual_seed(width)
    t, k, eps, alpha = 19, 3, 1e-5, 1.7
    x, gain = torch.randn(t, width, generator=g) * 2, 1 + 0.3 * torch.randn(width, generator=g)
    y = (torch.randn(t * k, width, generator=g) * 3).to(dtype)
    wts = torch.rand(t, k, generator=g)
    ga, gb = 1 + 0.5 * torch.randn(width, generator=g), 1 + 0.5 * torch.randn(width, generator=g)
    a, b = y[:t].contiguous(), (y[t:2 * t] * 0.01).contiguous()

    def want(add):
        return plain.rms_norm(alpha * x.double() + add, gain, eps)
    cases = [(want(a.double()), dict(y=a.to(DEV))),
             (want((y.double().view(t, k, width) * wts.double()[:, :, None]).sum(1)),
              dict(y=y.to(DEV), weights=wts.to(DEV))),
             (want(0.5 * (plain.rms_norm(a.double(), ga, eps) + plain.rms_norm(b.double(), gb, eps))),
              dict(y=NormedSum(a.to(DEV), ga.to(DEV), b.to(DEV), gb.to(DEV), eps, 0.5)))]
    for ref, kw in cases:
        res, out = x.to(DEV), torch.empty(t, width, dtype=dtype, device=DEV)
        ops.post_norm(res, gain=gain.to(DEV), eps=eps, alpha=alpha, out=out, **kw)
        assert rel_err(res, ref) < 2e-6
        assert torch.equal(out, res.to(dtype))
        res = x.to(DEV)
        ops.post_norm(res, gain=gain.to(DEV), eps=eps, alpha=alpha, **kw)
        assert rel_err(res, ref) < 2e-6


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_head_norm_without_a_gate(ops, dtype):
    g = torch.Generator().manual_seed(1)
    t, heads, vdim = 21, 3, 20
    o, w = torch.randn(t, heads * vdim, generator=g), 1 + 0.3 * torch.randn(vdim, generator=g)
    out = torch.empty(t, heads * vdim, dtype=dtype, device=DEV)
    ops.gated_rmsnorm(o.to(DEV), None, w.to(DEV), 1e-5, out, group=vdim)
    ref = plain.rms_norm(o.double().view(t, heads, vdim), w, 1e-5).reshape(t, -1)
    assert rel_err(out, ref) < (2e-6 if dtype == torch.float32 else 5e-3)


def _gather(pool, table, n, page_size):
    """Rows 0 .. n - 1 of a request from its pages: [n, heads, numbers]."""
    js = torch.arange(n)
    pages = table[js // page_size].long()
    return pool[pages, :, js % page_size, :]


def _tables(counts, spare, g):
    """Shuffled page numbers for each request: (lists of pages, pages in all)."""
    total = sum(counts) + spare
    perm = torch.randperm(total, generator=g).tolist()
    return [[perm.pop() for _ in range(n)] for n in counts], total


def _rows(tables, who, width):
    return torch.tensor([tables[r] + [-1] * (width - len(tables[r])) for r in who], dtype=torch.int32, device=DEV)


@pytest.mark.parametrize("dtype,plain_kernel", KERNELS, indirect=["plain_kernel"])
@pytest.mark.parametrize("heads,kv,dim,vdim,rot,pairing,pool,temp,rows", [
    (6, 3, 20, 20, 10, "interleaved", 3, False, 1), (4, 2, 64, 64, 64, "interleaved", 8, False, 1),
    (8, 2, 64, 32, 32, "half", None, True, 1), (2, 1, 88, 72, 40, "half", None, True, 1), (3, 1, 36, 36, 36, "interleaved", 7, True, 1),
    (2, 2, 16, 16, 0, "half", 1, False, 1), (1, 1, 8, 40, 8, "half", 5, True, 1), (16, 4, 128, 128, 128, "interleaved", 16, False, 16),
    (16, 4, 128, 128, 64, "half", 16, True, 16), (40, 8, 256, 256, 32, "half", None, False, 16), (5, 1, 128, 128, 12, "interleaved", 4, False, 16)])
def test_projected_rows_on_their_way_to_attention(ops, dtype, plain_kernel, heads, kv, dim, vdim, rot, pairing, pool, temp, rows):
    """Whole-projection norms, a rotation with a magnitude, the factor per head, the cache write
    (values of their own or the keys' own columns) and the means of completed blocks: three
    requests in portions down to two rows and single rows, with the projected rows as columns
    of a wider tensor, against the plain functions on the whole request. `rows`: how many times
    as long the requests are (many rows take kernels of their own)."""
    g = torch.Generator().manual_seed(dim + heads)
    lens, ps, bps, eps = [45 * rows, 7, 30 * rows], 8, 4, 1e-5
    keys_are_values = vdim == dim
    nq, nk, nv = heads * dim, kv * dim, kv * vdim
    ch = nq + nk + (0 if keys_are_values else nv)
    v_col = nq if keys_are_values else nq + nk
    u_all = [(torch.randn(n, ch, generator=g) * 1.5).to(dtype) for n in lens]
    qn, kn = 1 + 0.3 * torch.randn(nq, generator=g), 1 + 0.3 * torch.randn(nk, generator=g)
    hs = 1 + 0.5 * torch.randn(heads, generator=g) if temp else None
    r = rudazen_cases.rot(rot, 300.0, (3.0, 40, 4.0, 0.5))
    freq, mag = plain.frequencies(r) if rot else (None, 1.0)
    tables, pages = _tables([-(-n // ps) for n in lens], 2, g)
    k_pool = torch.full((pages, kv, ps, dim), float("nan"), dtype=dtype, device=DEV)
    v_pool = torch.full((pages, kv, ps, vdim), float("nan"), dtype=dtype, device=DEV)
    if pool:
        from ninfer_amd.parts import CacheView
        btables, bpages = _tables([-(-(n // pool) // bps) for n in lens], 2, g)
        blk = {"k_block": torch.full((bpages, kv, bps, dim), float("nan"), dtype=dtype, device=DEV),
               "v_block": torch.full((bpages, kv, bps, vdim), float("nan"), dtype=dtype, device=DEV)}
    got_q = [torch.zeros(n, nq) for n in lens]
    cuts = [_cut(lens[0], [13, 2, (9 if rows == 1 else 36 * rows + 1), 3], 6), _cut(7, [3, 2], 2), _cut(lens[2], [2, 11 * rows, 1, 8], 4)]
    for ctx, who, starts, counts in _steps(ops, dtype, cuts, [0, 1, 2]):
        wide = torch.zeros(ctx.T, ch + 24, dtype=dtype, device=DEV)
        wide[:, 8:8 + ch] = torch.cat([u_all[i][s:s + n] for i, s, n in zip(who, starts, counts)]).to(DEV)
        q = torch.empty(ctx.T, nq, dtype=dtype, device=DEV)
        blocks = None
        if pool:
            blocks = CacheView(blk, _rows(btables, who, max(1, max(len(t) for t in btables))), bps, None, stride=pool)
        ops.qkv_wide(wide[:, 8:8 + ch], ctx, q, heads, kv, dim, vdim, k_pool, v_pool,
                     _rows(tables, who, max(len(t) for t in tables)), ps, v_col=v_col, q_norm=qn.to(DEV),
                     k_norm=kn.to(DEV), norm_eps=eps, inv_freq=freq.float().to(DEV) if rot else None, rot_dim=rot,
                     interleaved=pairing == "interleaved", magnitude=mag, head_scale=hs.to(DEV) if temp else None,
                     blocks=blocks)
        o = 0
        for i, s, n in zip(who, starts, counts):
            got_q[i][s:s + n] = q[o:o + n].float().cpu()
            o += n
    # (a 32-bit angle of hundreds of radians is off by some 1e-5)
    tol = (3e-6 if rows == 1 else 1e-5) if dtype == torch.float32 else 6e-3
    for i, n in enumerate(lens):
        x, pos = u_all[i].double(), torch.arange(n)
        q = plain.rotate(plain.rms_norm(x[:, :nq], qn, eps).reshape(n, heads, dim), pos, r if rot else None, pairing)
        if temp:
            q = q * hs.double()[None, :, None]
        assert rel_err(got_q[i], q.reshape(n, -1)) < tol
        k = plain.rotate(plain.rms_norm(x[:, nq:nq + nk], kn, eps).reshape(n, kv, dim), pos, r if rot else None, pairing)
        table = torch.tensor(tables[i])
        have_k, have_v = _gather(k_pool.cpu(), table, n, ps), _gather(v_pool.cpu(), table, n, ps)
        assert rel_err(have_k, k) < tol
        assert torch.equal(have_v, u_all[i][:, v_col:v_col + nv].reshape(n, kv, vdim))
        if pool and n >= pool:
            # the means of what the pages hold, rounded once
            for name, have in (("k_block", have_k), ("v_block", have_v)):
                mean = plain.block_means(have.double(), pool)
                got = _gather(blk[name].cpu(), torch.tensor(btables[i]), n // pool, bps)
                assert rel_err(got, mean) < (1e-6 if dtype == torch.float32 else 3e-3)
                assert (got.double() - mean).abs().max() <= (1e-6 if dtype == torch.float32 else 2.0 ** -8) * mean.abs().max()


class _Cached:
    """Keys and values of a few requests laid into shuffled pages, and the means of their blocks."""

    def __init__(self, lens, kv, dim, vdim, ps, dtype, g, pool=None, bps=4, spare=3):
        self.ps, self.bps, self.lens, self.pool, self.dtype = ps, bps, lens, pool, dtype
        self.k = [torch.randn(n, kv, dim, generator=g).to(dtype) for n in lens]
        self.v = [torch.randn(n, kv, vdim, generator=g).to(dtype) for n in lens]
        self.shape = (kv, dim, vdim)
        self.tables, self.pages = _tables([-(-n // ps) for n in lens], spare, g)
        if pool:
            self.btables, self.bpages = _tables([-(-(n // pool) // bps) for n in lens], spare, g)

    def _lay(self, rows, tables, pages, ps):
        pool = torch.full((pages, rows[0].shape[1], ps, rows[0].shape[2]), float("nan"), dtype=self.dtype)
        for r, x in enumerate(rows):
            js = torch.arange(x.shape[0])
            if len(js):
                pool[torch.tensor(tables[r])[js // ps], :, js % ps] = x
        return pool.to(DEV)

    def lay(self):
        k, v = self._lay(self.k, self.tables, self.pages, self.ps), self._lay(self.v, self.tables, self.pages, self.ps)
        if self.pool:
            # (rounded as the cache rounds them; `means` is what the attention sees)
            self.km = [plain.block_means(x.double(), self.pool).to(self.dtype) for x in self.k]
            self.vm = [plain.block_means(x.double(), self.pool).to(self.dtype) for x in self.v]
            self.blk = {"k_block": self._lay(self.km, self.btables, self.bpages, self.bps),
                        "v_block": self._lay(self.vm, self.btables, self.bpages, self.bps)}
        return k, v

    def table(self, who, lo):
        """Block table rows of the requests `who`, the pages wholly before position lo[i] given
        as -1, as a window's cache gives them back."""
        rows = []
        width = max(len(t) for t in self.tables)
        for i, r in enumerate(who):
            t = list(self.tables[r]) + [-1] * (width - len(self.tables[r]))
            for p in range(max(lo[i], 0) // self.ps):
                t[p] = -1
            rows.append(t)
        return torch.tensor(rows, dtype=torch.int32, device=DEV)

    def blocks(self, who, upto, window):
        """The view of the blocks; the pages of blocks no row sees yet are given as -1 (upto[i]:
        the last position of request i in the step)."""
        if not self.pool:
            return None
        from ninfer_amd.parts import CacheView
        width = max(1, max(len(t) for t in self.btables))
        rows = []
        for i, r in enumerate(who):
            seen = max(0, (upto[i] - window + 1) // self.pool)
            t = list(self.btables[r]) + [-1] * (width - len(self.btables[r]))
            rows.append([p if j * self.bps < seen else -1 for j, p in enumerate(t)])
        return CacheView(self.blk, torch.tensor(rows, dtype=torch.int32, device=DEV), self.bps, None, stride=self.pool)


def _dense_attention(q, c, r, heads, kv, window, scale, gate=None):
    """The plain softmax of q [n, heads, d] over request r of the cache, with the block means as
    the cache holds them."""
    n, per = q.shape[0], heads // kv
    k, v, vis = c.k[r].double(), c.v[r].double(), plain.visible(n, window)
    if c.pool:
        k, v = torch.cat([c.km[r].double(), k]), torch.cat([c.vm[r].double(), v])
        vis = torch.cat([plain.visible_blocks(n, window, c.pool), vis], 1)
    out = torch.zeros(n, heads, v.shape[-1], dtype=D)
    for a in range(heads):
        s = q[:, a].double() @ k[:, a // per].T * scale
        out[:, a] = torch.softmax(torch.where(vis, s, torch.full((), -math.inf, dtype=D)), -1) @ v[:, a // per]
    out = out.reshape(n, -1)
    return out if gate is None else out * torch.sigmoid(gate.double())


SHAPES = [  # heads, kv, dim, vdim, window, pool, page, page of blocks
    (6, 3, 20, 20, 10, 3, 4, 4), (8, 2, 64, 64, 32, 8, 16, 16), (4, 4, 32, 96, 48, 1, 8, 8), (6, 2, 88, 72, 52, 5, 16, 2),
    (16, 2, 64, 32, 16, 2, 16, 8), (3, 1, 128, 128, 70, 4, 32, 32), (2, 2, 8, 24, None, None, 8, 4), (5, 5, 40, 8, 1, 1, 2, 2),
    (40, 1, 16, 16, 9, 2, 4, 16), (4, 1, 128, 128, 64, 2, 16, 16), (16, 4, 64, 64, 24, 1, 8, 8), (8, 2, 128, 128, 40, None, 16, 16),
    (6, 1, 128, 128, 17, 1, 16, 16), (2, 2, 128, 128, 33, 3, 64, 64)]


@pytest.mark.parametrize("dtype,plain_kernel", KERNELS, indirect=["plain_kernel"])
@pytest.mark.parametrize("gated", [True, False])
@pytest.mark.parametrize("heads,kv,dim,vdim,window,pool,ps,bps", SHAPES)
def test_attention_with_blocks_and_gate(ops, dtype, plain_kernel, gated, heads, kv, dim, vdim, window, pool, ps, bps):
    """Three requests: whole prompts in one step, then a step that mixes single rows with a
    portion, then single rows alone (the kernels for prompt tiles and for single rows, and the
    plain kernel), pages before the window given back, pages of blocks not yet seen absent;
    against the plain softmax."""
    g = torch.Generator().manual_seed(heads * dim + (window or 0))
    lens = [310, 37, 141]
    c = _Cached(lens, kv, dim, vdim, ps, dtype, g, pool, bps)
    k_pool, v_pool = c.lay()
    q = [torch.randn(n, heads, dim, generator=g).to(dtype) for n in lens]
    gate = [torch.randn(n, heads * vdim, generator=g).to(dtype) if gated else None for n in lens]
    scale = 0.9 / math.sqrt(dim)
    want = [_dense_attention(q[r], c, r, heads, kv, window, scale, gate[r]) for r in range(3)]
    tol = 2e-5 if dtype == torch.float32 else 1.2e-2
    # (request, first row, rows) of every step; single rows first
    for step in ([(0, 0, 310), (1, 0, 37), (2, 0, 141)], [(1, 36, 1), (2, 69, 1), (0, 97, 213)],
                 [(0, 309, 1), (1, 20, 1), (2, 64, 1)], [(2, 3, 2), (0, 60, 33)], [(0, 200, 1)]):
        ctx = util.make_context(ops, dtype, [(s, n) for _, s, n in step])
        ctx.single_rows = sum(1 for _, _, n in step if n == 1) if step[0][2] == 1 else 0
        who = [r for r, _, _ in step]
        bt = c.table(who, [s - window + 1 if window else 0 for _, s, _ in step])
        rows = torch.cat([q[r][s:s + n] for r, s, n in step]).reshape(ctx.T, heads * dim).to(DEV)
        wide = None
        if gated:
            wide = torch.zeros(ctx.T, heads * vdim + 16, dtype=dtype, device=DEV)
            wide[:, 8:8 + heads * vdim] = torch.cat([gate[r][s:s + n] for r, s, n in step]).to(DEV)
            wide = wide[:, 8:8 + heads * vdim]
        out = torch.full((ctx.T, heads * vdim), float("nan"), dtype=dtype, device=DEV)
        ops.paged_attention(rows, k_pool, v_pool, bt, ctx, heads, kv, dim, ps, window, scale, out, vdim=vdim,
                            blocks=c.blocks(who, [s + n - 1 for _, s, n in step], window), gate=wide)
        ref = torch.cat([want[r][s:s + n] for r, s, n in step]).reshape(ctx.T, -1)
        assert torch.isfinite(out).all()
        assert rel_err(out, ref) < tol, step


@pytest.mark.parametrize("dtype,plain_kernel", KERNELS, indirect=["plain_kernel"])
@pytest.mark.parametrize("dim", [32, 128])
@pytest.mark.parametrize("window,pool,ps", [(44, 8, 16), (64, 16, 16), (17, 5, 8), (24, 1, 16)])
def test_one_loud_key_and_one_loud_block_at_the_edges(ops, dtype, plain_kernel, dim, window, pool, ps):
    """Among hundreds of quiet keys one block of keys whose mean's score stands out, with a value
    no other key has. The block just seen, and one that is not yet seen because its last token
    is still inside the window (or has just left it with the block's last token one position
    too late); one loud key just inside the window, and just outside, where only its block's
    mean (a `pool`-th of it) may be seen. For a row inside a prompt portion and for one decoded
    alone; blocks far back and at a tile's and page's border of blocks."""
    heads, kv, vdim, n = 4, 1, dim, 700
    g = torch.Generator().manual_seed(7)
    for row in (699, 640, 575, 301, 256, window + pool - 1, window + 2 * pool):
        seen = (row - window + 1) // pool
        places = [("in", b) for b in {seen - 1, 0, min(63, seen - 1), min(64, seen - 1)} if 0 <= b < seen] + [("out", seen)]
        places += [("key", row - window + 1), ("left", row - window)]
        for what, at in places:
            c = _Cached([n], kv, dim, vdim, ps, dtype, g, pool, bps=16)
            c.k[0] *= 0.05
            c.v[0] *= 0.1
            if what in ("in", "out"):
                # loud keys only outside the window: what is inside stays quiet
                js = [j for j in range(at * pool, at * pool + pool) if j <= row - window]
                if what == "out" and not js:
                    continue
            else:
                js = [at]
            c.k[0][js, :, 0] = 30.0
            c.v[0][js] = 5.0
            q = (torch.randn(n, heads, dim, generator=g) * 0.05).to(dtype)
            q[row, :, 0] = 30.0
            k_pool, v_pool = c.lay()
            ref = _dense_attention(q[:row + 1], _Sub(c, row + 1), 0, heads, kv, window, 0.2)[row]
            if what in ("in", "key"):
                assert (ref - 5.0).abs().max() < 1e-6
            elif what == "out":
                assert ref.abs().max() < 0.3
            for first, count in ((row - min(row, 37), min(row, 37) + 1), (row, 1)):
                ctx = util.make_context(ops, dtype, [(first, count)])
                ctx.single_rows = 1 if count == 1 else 0
                out = torch.empty(count, heads * vdim, dtype=dtype, device=DEV)
                ops.paged_attention(q[first:first + count].reshape(count, -1).to(DEV), k_pool, v_pool,
                                    c.table([0], [first - window + 1]), ctx, heads, kv, dim, ps, window, 0.2, out,
                                    vdim=vdim, blocks=c.blocks([0], [row], window))
                assert (out[-1].double().cpu() - ref).abs().max() < (1e-4 if dtype == torch.float32 else 0.05), (row, what, at, count)


class _Sub:
    """The first n positions of a one-request cache."""

    def __init__(self, c, n):
        self.pool, nb = c.pool, n // c.pool
        self.k, self.v, self.km, self.vm = [c.k[0][:n]], [c.v[0][:n]], [c.km[0][:nb]], [c.vm[0][:nb]]


@pytest.mark.parametrize("dtype,plain_kernel", KERNELS, indirect=["plain_kernel"])
@pytest.mark.parametrize("heads,dim,vdim,rows", [(3, 12, 20, 1), (2, 64, 128, 1), (1, 4, 8, 1), (4, 20, 9, 1), (2, 128, 64, 1),
                                                 (2, 64, 128, 12), (3, 32, 40, 9)])
def test_recurrence_with_a_forget_gate(ops, dtype, plain_kernel, heads, dim, vdim, rows):
    """Three requests in slots 2, 0 and 3 of a wider state tensor, cut into portions down to two
    rows and single rows, with gates from nearly shut to nearly open and lower bounds of 0, in
    between, and 1 (nothing is ever written), against the plain recurrence of the whole request."""
    g = torch.Generator().manual_seed(dim + vdim)
    lens = [45 * rows, 7, 30 * rows]
    n = heads * dim
    ch = 2 * n + heads * vdim
    u_all = []
    for ln in lens:
        u = torch.randn(ln, ch, generator=g)
        u[:, n:2 * n] *= 6.0
        u_all.append(u.to(dtype))
    bias, lower = torch.randn(n, generator=g) * 2, torch.rand(n, generator=g)
    lower[0], lower[1] = 0.0, 1.0
    floats = heads * dim * vdim
    state = torch.full((4, floats + 9), 7.0, device=DEV)
    state[:, 4:4 + floats] = 0
    got = [torch.zeros(ln, heads * vdim) for ln in lens]
    cuts = [_cut(lens[0], [13, 2, 9 * rows, 3], 6), _cut(7, [3, 2], 2), _cut(lens[2], [2, 11 * rows, 1, 8], 4)]
    for ctx, who, starts, counts in _steps(ops, dtype, cuts, [2, 0, 3]):
        wide = torch.zeros(ctx.T, ch + 11, dtype=dtype, device=DEV)
        wide[:, 3:3 + ch] = torch.cat([u_all[r][s:s + c] for r, s, c in zip(who, starts, counts)]).to(DEV)
        out = torch.empty(ctx.T, heads * vdim, device=DEV)
        wf = ops.gla_work_floats(dtype, ctx, heads, dim)
        work = torch.empty(ctx.T, wf, device=DEV) if wf else None
        ops.gated_linear_attention(wide[:, 3:3 + ch], 0, 0, 2 * n, None, heads, dim, vdim, 1.0, 1.0,
                                   state[:, 4:4 + floats], ctx, out, work=work, forget=(n, bias.to(DEV), lower.to(DEV)))
        o = 0
        for r, s, c in zip(who, starts, counts):
            got[r][s:s + c] = out[o:o + c].cpu()
            o += c
    for r, (ln, slot) in enumerate(zip(lens, [2, 0, 3])):
        u = u_all[r].double()
        q = plain.silu(u[:, :n]).view(ln, heads, dim)
        f = plain.forget_gates(u[:, n:2 * n] + bias.double(), lower).view(ln, heads, dim)
        o, last = plain.gated_recurrence(q, f, u[:, 2 * n:].reshape(ln, heads, vdim))
        assert rel_err(got[r], o.reshape(ln, -1)) < 1e-5
        assert rel_err(state[slot, 4:4 + floats], last.reshape(-1)) < 1e-5
    assert (state[:, :4] == 7).all() and (state[:, 4 + floats:] == 7).all() and (state[1, 4:4 + floats] == 0).all()


@pytest.mark.parametrize("lens,first", [([300, 129, 700], 0), ([128, 1, 640], 5), ([513], 2), ([256, 257], 16)])
def test_recurrence_in_long_portions_of_several_requests(ops, lens, first):
    """Long portions side by side, each after `first` rows in a step before: pieces of a request
    that the kernels work on side by side, whole ones and short last ones, a request that is
    shorter than a piece; the state they leave, and one more row after it."""
    heads, dim, vdim = 2, 20, 24
    g = torch.Generator().manual_seed(sum(lens))
    n = heads * dim
    total = [first + ln + 1 for ln in lens]
    u_all = [torch.randn(t, 2 * n + heads * vdim, generator=g).to(torch.bfloat16) for t in total]
    bias, lower = torch.randn(n, generator=g) + 2, torch.rand(n, generator=g)
    state = torch.zeros(len(lens), heads * dim * vdim, device=DEV)
    got = [torch.zeros(t, heads * vdim) for t in total]
    cuts = [([first] if first else []) + [ln, 1] for ln in lens]
    slots = list(range(len(lens)))[::-1]
    for ctx, who, starts, counts in _steps(ops, torch.bfloat16, cuts, slots):
        u = torch.cat([u_all[r][s:s + c] for r, s, c in zip(who, starts, counts)]).to(DEV)
        out = torch.empty(ctx.T, heads * vdim, device=DEV)
        wf = ops.gla_work_floats(torch.bfloat16, ctx, heads, dim)
        work = torch.empty(ctx.T, wf, device=DEV) if wf else None
        ops.gated_linear_attention(u, 0, 0, 2 * n, None, heads, dim, vdim, 1.0, 1.0, state, ctx, out, work=work,
                                   forget=(n, bias.to(DEV), lower.to(DEV)))
        o = 0
        for r, s, c in zip(who, starts, counts):
            got[r][s:s + c] = out[o:o + c].cpu()
            o += c
    assert ops.lib.ninfer_gla_segment_floats(sum(lens), len(lens), heads, dim, vdim) > 0
    for r, t in enumerate(total):
        u = u_all[r].double()
        f = plain.forget_gates(u[:, n:2 * n] + bias.double(), lower).view(t, heads, dim)
        o, last = plain.gated_recurrence(plain.silu(u[:, :n]).view(t, heads, dim), f, u[:, 2 * n:].reshape(t, heads, vdim))
        assert rel_err(got[r], o.reshape(t, -1)) < 1e-5
        assert rel_err(state[slots[r]], last.reshape(-1)) < 1e-5


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_recurrence_remembers_and_forgets(ops, dtype):
    """A loud token hundreds of rows back: a channel whose gate is all but open keeps it to the
    end, one that is all but shut has nothing of it left a row later; in a prompt of one piece,
    in portions and token by token."""
    heads, dim, vdim, n = 1, 4, 16, 600
    ch = 2 * dim + vdim
    u = torch.zeros(n, ch)
    u[:, 0:2] = 3.0                                  # q reads channels 0 and 1
    u[:, dim] = 14.0                                 # channel 0: f = 1 - 8e-7
    u[:, dim + 1] = -14.0                            # channel 1: f = 8e-7
    u[3, dim] = 0.0                                  # ... except here, where half is written
    u[3, 2 * dim:] = 100.0
    u = u.to(dtype)
    f = plain.forget_gates(u[:, dim:2 * dim].double(), torch.zeros(dim)).view(n, heads, dim)
    want, _ = plain.gated_recurrence(plain.silu(u[:, :dim].double()).view(n, heads, dim), f,
                                     u[:, 2 * dim:].double().view(n, heads, vdim))
    assert abs(float(want[-1, 0, 0]) - 0.5 * 100 * float(plain.silu(torch.tensor(3.0, dtype=D)))) < 0.5
    for cut in ([n], [257, 2, 341], _cut(n, [590], 10)):
        state, got = torch.zeros(1, dim * vdim, device=DEV), []
        for ctx, _, starts, counts in _steps(ops, dtype, [cut], [0]):
            out = torch.empty(ctx.T, vdim, device=DEV)
            wf = ops.gla_work_floats(dtype, ctx, heads, dim)
            work = torch.empty(ctx.T, wf, device=DEV) if wf else None
            ops.gated_linear_attention(u[starts[0]:starts[0] + counts[0]].to(DEV), 0, 0, 2 * dim, None, heads, dim, vdim,
                                       1.0, 1.0, state, ctx, out, work=work,
                                       forget=(dim, torch.zeros(dim, device=DEV), torch.zeros(dim, device=DEV)))
            got.append(out.cpu())
        got = torch.cat(got)
        assert (got.double() - want[:, 0]).abs().max() < 1e-3 * want.abs().max()


# ---- whole models ----------------------------------------------------------------------------

PROMPT_LENGTHS = [70, 1, 23, 97, 40, 64]


def row_errors(got, ref):
    d = (got - ref).double()
    return (d - d.mean(-1, keepdim=True)).pow(2).mean(-1).sqrt() / ref.double().std()


def noise_of(cfg, w, toks, ref):
    """How far the plain implementation's logits move when every weight is disturbed by one
    part in 2^9 (what rounding to bfloat16 does to a number), several times for short requests
    (a row whose heads or sums all but cancel before a norm moves far in some draws only):
    median, ninth decile and largest of the rows' errors. The comparisons' bounds come from
    the model at hand."""
    g = torch.Generator().manual_seed(len(toks))
    errs = []
    for _ in range(6 if len(toks) <= 100 else 2):
        w2 = {k: v * (1 + torch.randn(v.shape, generator=g) * 2.0 ** -9) for k, v in w.items()}
        w2.update({k: v.clamp(0, 1) for k, v in w2.items() if k.endswith(".lower")})
        errs.append(row_errors(plain.forward(cfg, w2, toks)[0], ref))
    mid = torch.stack(errs).mean(0)
    return mid.median().item(), mid.kthvalue(max(1, int(0.9 * len(mid)))).values.item(), \
        torch.stack(errs).max().item()


@pytest.fixture(scope="module", params=list(rudazen_cases.CASES))
def case(request, tmp_path_factory):
    import ninfer_amd
    name = request.param
    make, seed = rudazen_cases.CASES[name]
    raw = make()
    out = {"name": name, "cfg": raw, "dirs": {}, "ref": {}, "noise": {},
           "reqs": {f"r{i}": util.random_tokens(n, raw["vocab"], 50 + i) for i, n in enumerate(PROMPT_LENGTHS)}}
    for dtype in ("float32", "bfloat16"):
        d = str(tmp_path_factory.mktemp(f"rudazen_{name}_{dtype}"))
        ninfer_amd.write_random_model(d, raw, seed, dtype=dtype, std=STD)
        out["dirs"][dtype] = d
        cfg, w = util.read_folder(d)
        out["ref"][dtype] = {k: plain.forward(cfg, w, v)[0] for k, v in out["reqs"].items()}
        out["noise"][dtype] = {k: noise_of(cfg, w, v, out["ref"][dtype][k]) for k, v in out["reqs"].items()}
    return out


def make_runner(case, dtype, page_size=8, num_pages=40, seqs=4, **more):
    from ninfer_amd import EngineOptions, load_model
    opt = EngineOptions(dtype=dtype, max_context=128, num_sequences=seqs, page_size=page_size,
                        num_pages=num_pages, check_pages=True, poison_freed_pages=True, **more)
    return load_model(case["dirs"][dtype], opt)


def check_logits(case, dtype, got, what):
    for rid, g in got.items():
        ref = case["ref"][dtype][rid]
        who = f"{case['name']} {rid} {what}"
        assert g.shape == ref.shape, who
        assert torch.isfinite(g).all(), f"{who}: not finite"
        err = row_errors(g, ref)
        n50, n90, nmax = case["noise"][dtype][rid]
        f50, f90, fmax, floor = (3, 3, 3, 0.03) if dtype == "bfloat16" else \
            (8 * 2.0 ** -15, 8 * 2.0 ** -15, 16 * 2.0 ** -15, 3e-6)
        e50 = err.median().item()
        e90 = err.kthvalue(max(1, int(0.9 * len(err)))).values.item()
        if len(err) >= 20:
            assert e50 <= max(f50 * n50, floor), f"{who}: median row error {e50:.2e} (disturbance {n50:.2e})"
            assert e90 <= max(f90 * n90, floor), f"{who}: ninth decile {e90:.2e} (disturbance {n90:.2e})"
        assert err.max().item() <= max(fmax * nmax, 4 * floor), \
            f"{who}: row {err.argmax()} is off by {err.max():.2e} (disturbance {nmax:.2e})"


def test_layer_by_layer(case):
    """The 32-bit residual stream after every layer, for a prompt in one step and in portions."""
    from ninfer_amd.engine import Chunk
    cfg, w = util.read_folder(case["dirs"]["float32"])
    toks = case["reqs"]["r4"]
    streams = plain.forward(cfg, w, toks)[1]
    runner = make_runner(case, "float32")
    assert len(runner.spec.plan) == len(streams)
    for cuts in ([len(toks)], [17, 2, len(toks) - 19]):
        slot = runner.open()
        got = [[] for _ in streams]
        runner.tap = lambda i, residual, pending: got[i].append(residual.cpu().clone())
        o = 0
        for n in cuts:
            runner.step([Chunk(slot, toks[o:o + n], [])])
            o += n
        runner.tap = None
        runner.close(slot)
        for i, want in enumerate(streams):
            g = torch.cat(got[i]).double()
            assert (g - want).abs().max() <= 2e-5 * max(1.0, want.abs().max().item()), f"layer {i}"


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_whole_tail_portions(case, dtype):
    runner = make_runner(case, dtype)
    for rid, toks in case["reqs"].items():
        for what, sched in (("whole", util.schedule_whole(rid, toks)),
                            ("tail", util.schedule_tail(rid, toks, 48)),
                            ("portions", util.schedule_portions(rid, toks, seed=len(toks)))):
            if what == "tail" and len(toks) == 1:
                continue
            check_logits(case, dtype, util.run_schedule(runner, sched), what)
    runner.cache.check()
    assert all(g.allocator.in_use == 0 for g in runner.cache.groups)


def test_cut_does_not_matter_in_32_bit(case):
    """Every way of cutting a request gives the same logits to the bit in 32-bit: all kernels
    of that path sum in an order that depends on the row alone."""
    runner = make_runner(case, "float32")
    toks = case["reqs"]["r3"]
    whole = util.run_schedule(runner, util.schedule_whole("a", toks))["a"]
    for sched in (util.schedule_tail("a", toks, 40), util.schedule_portions("a", toks, seed=3)):
        assert torch.equal(util.run_schedule(runner, sched)["a"], whole)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_mixed_batches_reuse_pages_and_slots(case, dtype):
    """Up to four live requests, prompt portions beside single tokens, in a pool so small that
    pages are used again (freed pages are filled with NaN) and with four state slots for twelve
    requests, then schedules drawn at random; every request's logits equal those of the
    request alone."""
    runner = make_runner(case, dtype, page_size=8, num_pages=34)
    reqs = dict(case["reqs"])
    reqs.update({k + "again": v for k, v in case["reqs"].items()})
    ref = {**case["ref"][dtype], **{k + "again": v for k, v in case["ref"][dtype].items()}}
    noise = {**case["noise"][dtype], **{k + "again": v for k, v in case["noise"][dtype].items()}}
    sub = {"name": case["name"], "ref": {dtype: ref}, "noise": {dtype: noise}}
    check_logits(sub, dtype, util.run_schedule(runner, util.schedule_mixed(reqs, seed=1)), "mixed")
    for seed in (2, 3):
        steps = util.schedule_random(reqs, seed)
        got = util.run_schedule(runner, steps)
        wanted = {}
        for entries, _ in steps:
            for rid, toks, want in entries:
                wanted.setdefault(rid, [0, []])
                wanted[rid][1] += [wanted[rid][0] + w_ for w_ in want]
                wanted[rid][0] += len(toks)
        part = {"name": case["name"], "noise": {dtype: noise},
                "ref": {dtype: {rid: ref[rid][rows] for rid, (_, rows) in wanted.items() if rows}}}
        check_logits(part, dtype, got, f"random {seed}")
    assert all(g.allocator.reused > 0 for g in runner.cache.groups)
    runner.cache.check()


def test_a_slot_used_again_starts_empty(case):
    """One state slot: every request gets the slot the last one left, with that request's
    recurrent state still in it unless it is cleared."""
    runner = make_runner(case, "float32", seqs=1)
    for rid in ("r3", "r0", "r1", "r2"):
        toks = case["reqs"][rid]
        sched = util.schedule_tail(rid, toks, 5) if len(toks) > 1 else util.schedule_whole(rid, toks)
        check_logits(case, "float32", util.run_schedule(runner, sched), "slot used again")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_decoding(case, dtype):
    """A few tokens of prompt, then hundreds of single steps: across pages, with every window
    passing over decoded tokens many times and giving its pages back, blocks completed by
    decoded tokens and seen a window later, across the attention kernels' tiles, with the
    recurrent state carried on."""
    if case["name"] == "ones" and dtype == "bfloat16":
        pytest.skip("covered by the other two")
    from ninfer_amd import EngineOptions, load_model
    n = 230
    cfg, w = util.read_folder(case["dirs"][dtype])
    toks = util.random_tokens(n, cfg["vocab"], 9)
    ref = plain.forward(cfg, w, toks)[0]
    runner = load_model(case["dirs"][dtype], EngineOptions(
        dtype=dtype, max_context=256, num_sequences=2, page_size=16, num_pages=18, check_pages=True,
        poison_freed_pages=True))
    got = util.run_schedule(runner, util.schedule_tail("x", toks, n - 3))["x"]
    sub = {"name": case["name"], "ref": {dtype: {"x": ref}}, "noise": {dtype: {"x": noise_of(cfg, w, toks, ref)}}}
    check_logits(sub, dtype, {"x": got}, "long decoding")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_long_prompt(case, dtype):
    """Hundreds of tokens in one step and in two portions (the kernels that many rows choose),
    with blocks far back and more of them than one tile holds."""
    from ninfer_amd import EngineOptions, load_model
    n = 600
    cfg, w = util.read_folder(case["dirs"][dtype])
    toks = util.random_tokens(n, cfg["vocab"], 19)
    ref = plain.forward(cfg, w, toks)[0]
    sub = {"name": case["name"], "ref": {dtype: {"x": ref}}, "noise": {dtype: {"x": noise_of(cfg, w, toks, ref)}}}
    runner = load_model(case["dirs"][dtype], EngineOptions(
        dtype=dtype, max_context=640, prefill_chunk=640, num_sequences=2, page_size=16, num_pages=40,
        check_pages=True, poison_freed_pages=True))
    check_logits(sub, dtype, util.run_schedule(runner, util.schedule_whole("x", toks)), "whole")
    steps = [([("x", toks[:557], list(range(557)))], []), ([("x", toks[557:], list(range(n - 557)))], ["x"])]
    check_logits(sub, dtype, util.run_schedule(runner, steps), "two portions")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_decoding_from_a_captured_graph(case, dtype):
    """Decode-only steps replayed from a HIP graph (the first step of a shape runs eagerly, the
    second is captured, the rest are replays), two requests side by side, every replay against
    the plain implementation: which tokens complete a block is decided on the device."""
    from ninfer_amd.engine import Chunk
    runner = make_runner(case, dtype, use_graph=True)
    reqs = {k: case["reqs"][k] for k in ("r0", "r4")}
    slots = {k: runner.open() for k in reqs}
    heads = {k: len(v) - 30 for k, v in reqs.items()}
    got = {k: [] for k in reqs}
    logits = runner.step([Chunk(slots[k], reqs[k][:heads[k]], list(range(heads[k]))) for k in reqs])
    o = 0
    for k in reqs:
        got[k].append(logits[o:o + heads[k]].float().cpu())
        o += heads[k]
    for i in range(30):
        logits = runner.step([Chunk(slots[k], [reqs[k][heads[k] + i]], [0]) for k in reqs])
        for j, k in enumerate(reqs):
            got[k].append(logits[j:j + 1].float().cpu().clone())
    assert len(runner._graphs) >= 1
    for k in reqs:
        runner.close(slots[k])
    check_logits(case, dtype, {k: torch.cat(v) for k, v in got.items()}, "graph replay")


@pytest.mark.parametrize("seed", list(range(10)))
def test_random_configurations(seed, tmp_path):
    """Configurations drawn at random (sizes, head counts, kinds and order of layers, windows,
    blocks, what is absent), in both precisions: whole, in portions and in a mixed batch."""
    import ninfer_amd
    from ninfer_amd import EngineOptions, load_model
    raw = rudazen_cases.random_config(seed)
    reqs = {f"q{i}": util.random_tokens(n, raw["vocab"], 7 * seed + i) for i, n in enumerate([33, 1, 14, 50])}
    for dtype in ("float32", "bfloat16"):
        d = str(tmp_path / dtype)
        ninfer_amd.write_random_model(d, raw, 100 + seed, dtype=dtype, std=STD)
        cfg, w = util.read_folder(d)
        ref = {k: plain.forward(cfg, w, v)[0] for k, v in reqs.items()}
        sub = {"name": f"random {seed}", "ref": {dtype: ref},
               "noise": {dtype: {k: noise_of(cfg, w, v, ref[k]) for k, v in reqs.items()}}}
        runner = load_model(d, EngineOptions(dtype=dtype, max_context=64, num_sequences=3, page_size=8,
                                             num_pages=20, check_pages=True, poison_freed_pages=True))
        for k, v in reqs.items():
            check_logits(sub, dtype, util.run_schedule(runner, util.schedule_whole(k, v)), "whole")
            check_logits(sub, dtype, util.run_schedule(runner, util.schedule_portions(k, v, seed=seed)), "portions")
        check_logits(sub, dtype, util.run_schedule(runner, util.schedule_mixed(reqs, seed=seed, max_live=3)), "mixed")
        runner.release()


def test_greedy_generation_through_the_scheduler(case):
    """The framework's own entry point: prompts of unequal length generated greedily by the
    scheduler (admission, portions under a token budget, batched decoding, sampling kernel),
    token for token what the plain implementation chooses."""
    from ninfer_amd import Ninfer, SamplingParams
    cfg, w = util.read_folder(case["dirs"]["float32"])
    prompts = [case["reqs"][k][:n] for k, n in (("r0", 19), ("r2", 3), ("r3", 41))]
    new = 10
    want = []
    for p in prompts:
        toks = list(p)
        for _ in range(new):
            z = plain.forward(cfg, w, toks)[0]
            top = torch.topk(z[-1], 2).values
            if top[0] - top[1] < 1e-3:
                break   # too close to call: the comparison ends here for this prompt
            toks.append(int(z[-1].argmax()))
        want.append(toks[len(p):])
    eng = Ninfer(case["dirs"]["float32"], max_context=128, prefill_chunk=16, num_sequences=2,
                 dtype="float32", page_size=8, num_pages=30)
    got = eng.generate(prompts, SamplingParams.greedy(new), stop_ids=[])
    eng.close()
    assert sum(len(x) for x in want) >= new
    assert [g[:len(x)] for g, x in zip(got, want)] == want


def test_command_line_and_trace_replay(case, tmp_path):
    """bin/trace_run on a model folder (a mixed schedule as JSON lines, the logits files
    against the plain implementation) and bin/ninfer generating greedily from it."""
    if case["name"] != "odd":
        pytest.skip("one configuration is enough for the programs")
    reqs = {k: case["reqs"][k] for k in ("r0", "r2", "r4", "r1")}
    steps = util.schedule_mixed(reqs, seed=4)
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    out_dir = str(tmp_path / "out")
    p = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model",
                        case["dirs"]["float32"], "--dtype", "float32", "--out", out_dir,
                        "--max-tokens", "256"], input=util.write_trace(steps), text=True,
                       capture_output=True, timeout=600)
    assert p.returncode == 0, p.stderr[-2000:]
    assert [l for l in p.stdout.splitlines() if l.startswith("done ")] == [f"done {i}" for i in range(len(steps))]
    got = util.read_trace_output(out_dir, steps, case["cfg"]["vocab"])
    check_logits(case, "float32", got, "trace_run")
    stats = json.load(open(os.path.join(out_dir, "stats.json")))
    assert all(g["in_use"] == 0 for g in stats["groups"]) and any(g["window_freed"] > 0 for g in stats["groups"])
    prompt = case["reqs"]["r2"][:9]
    p = subprocess.run([sys.executable, os.path.join(root, "bin", "ninfer"), case["dirs"]["float32"], "--dtype",
                        "float32", "--prompt-ids", ",".join(map(str, prompt)), "--max-new", "4", "--temperature",
                        "0", "--max-context", "64"], text=True, capture_output=True, timeout=600)
    assert p.returncode == 0, p.stderr[-2000:]
    cfg, w = util.read_folder(case["dirs"]["float32"])
    first = int(plain.forward(cfg, w, prompt)[0][-1].argmax())
    assert str(first) in p.stdout
