"""Nosedra on the GPU against the plain implementation: every mechanism alone through its
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

import nosedra_cases
import plain_nosedra as plain
import util

pytestmark = pytest.mark.gpu
DEV = "cuda"
STD = 0.25
D = torch.float64
BOTH = [torch.float32, torch.bfloat16]
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


def _columns(x, pad):
    """The same numbers as columns of a wider tensor, `pad` columns in front and behind."""
    wide = torch.zeros(x.shape[0], x.shape[1] + 2 * pad, dtype=x.dtype, device=DEV)
    wide[:, pad:pad + x.shape[1]] = x.to(DEV)
    return wide[:, pad:pad + x.shape[1]]


# ---- mechanisms alone ------------------------------------------------------------------------

@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("width", [70, 256, 1100, 5000])
def test_stream_between_sublayers(ops, dtype, width):
    """What is added to the stream (nothing, rows, two rows with factors, rows with a bias, rows
    normed by themselves), formed in 32-bit, and the stream handed on normed or as it is; for
    all rows and for selected ones, which leave the stream alone."""
    from ninfer_amd.parts import NormedRows, SumRows
    g = torch.Generator().manual_seed(width)
    t, eps = 19, 1e-5
    x, w = torch.randn(t, width, generator=g) * 2, 0.3 * torch.randn(width, generator=g)
    a, b = ((torch.randn(t, width, generator=g) * 3).to(dtype) for _ in range(2))
    bias, gain = torch.randn(width, generator=g), 1 + 0.5 * torch.randn(width, generator=g)
    small = (a * 0.001).contiguous()    # (eps counts)
    da, db = a.to(DEV), b.to(DEV)
    cases = [(None, 0.0), (da, a.double()),
             (SumRows(da, 0.7, db, -1.3), 0.7 * a.double() - 1.3 * b.double()),
             (SumRows(da, bias=bias.to(DEV)), a.double() + bias.double()),
             (NormedRows(small.to(DEV), gain.to(DEV), eps), plain.unit(small.double(), eps) * gain.double())]
    rows = torch.tensor([3, 18, 0], dtype=torch.int32, device=DEV)
    tol = 2e-6 if dtype == torch.float32 else 4e-3
    for pending, add in cases:
        z = x.double() + add
        for normed in (True, False):
            want = plain.offset_norm(z, w, eps) if normed else z
            kw = dict(gain=(1 + w).to(DEV), eps=eps) if normed else {}
            res, out = x.to(DEV), torch.empty(t, width, dtype=dtype, device=DEV)
            ops.stream_norm(res, pending, out=out, **kw)
            assert rel_err(res, z) < 1e-6 and rel_err(out, want) < tol
            res, out = x.to(DEV), torch.empty(3, width, dtype=dtype, device=DEV)
            ops.stream_norm(res, pending, out=out, rows=rows, **kw)
            assert torch.equal(res.cpu(), x) and rel_err(out, want[[3, 18, 0]]) < tol
        res = x.to(DEV)
        if pending is not None:
            ops.stream_norm(res, pending)
            assert rel_err(res, z) < 1e-6


@pytest.mark.parametrize("dtype", BOTH)
def test_token_gate(ops, dtype):
    g = torch.Generator().manual_seed(3)
    t, d, layers, vocab = 37, 9, 4, 50
    z, table = (torch.randn(t, d, generator=g) * 2).to(dtype), torch.randn(vocab, layers * d, generator=g).to(dtype)
    toks = torch.randint(0, vocab, (t,), generator=g)
    for layer in (0, 3):
        out = torch.empty(t, d, dtype=dtype, device=DEV)
        ops.token_gate(z.to(DEV), table.to(DEV), toks.int().to(DEV), layer * d, out)
        want = plain.gelu(z.double()) * table.double()[toks][:, layer * d:(layer + 1) * d]
        assert rel_err(out, want) < (1e-6 if dtype == torch.float32 else 4e-3)


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("channels,taps,lens", [(37, 4, [45, 7, 30]), (96, 4, [700, 3, 61]), (64, 1, [20, 5, 9]),
                                                (40, 2, [310, 300, 2]), (24, 3, [280, 9, 33]), (16, 6, [290, 4, 12]),
                                                (8, 9, [20, 7, 3])])
def test_convolution_with_silu(ops, dtype, channels, taps, lens):
    """Three requests in portions down to two rows (shorter than the taps) and single rows, the
    inputs as columns of a wider tensor, the state in slots of a wider one."""
    g = torch.Generator().manual_seed(channels + taps)
    w, b = torch.randn(channels, taps, generator=g), torch.randn(channels, generator=g)
    xs = [torch.randn(n, channels, generator=g).to(dtype) for n in lens]
    state = torch.zeros(4, (taps - 1) * channels + 8, device=DEV)
    got = [torch.zeros(n, channels) for n in lens]
    cuts = [_cut(n, [2, max(n // 2, 2), 3, 5], min(4, n - 2)) for n in lens]
    slots = [2, 0, 3]
    for ctx, who, starts, counts in _steps(ops, dtype, cuts, slots):
        u = _columns(torch.cat([xs[r][s:s + n] for r, s, n in zip(who, starts, counts)]), 8)
        out = torch.empty(ctx.T, channels, dtype=dtype, device=DEV)
        ops.conv_silu(u, w.t().contiguous().to(DEV), b.to(DEV), state[:, 4:-4] if taps > 1 else None, ctx, out)
        o = 0
        for r, s, n in zip(who, starts, counts):
            got[r][s:s + n] = out[o:o + n].float().cpu()
            o += n
    for r, n in enumerate(lens):
        want = plain.silu(plain.causal_conv(xs[r].double(), w, b))
        assert rel_err(got[r], want) < (2e-6 if dtype == torch.float32 else 4e-3)
        if taps > 1:
            last = torch.cat([torch.zeros(taps - 1, channels), xs[r].float()])[-(taps - 1):]
            assert torch.equal(state[slots[r], 4:-4].cpu(), last.reshape(-1))
    assert (state[1] == 0).all() and (state[:, :4] == 0).all() and (state[:, -4:] == 0).all()


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("heads,dim", [(3, 20), (6, 64), (2, 700), (1, 2048), (4, 2048), (33, 8)])
def test_gated_norm_in_its_forms(ops, dtype, heads, dim):
    """The gate behind the norm or in front of it, the norm over a row, its equal parts or every
    head, one weight per column, and a divisor per head."""
    g = torch.Generator().manual_seed(heads * dim)
    t, n, eps = 11, heads * dim, 1e-5
    o, w = torch.randn(t, n, generator=g) * 0.01, 1 + 0.3 * torch.randn(n, generator=g)
    gate, den = torch.randn(t, n, generator=g).to(dtype), 0.02 + torch.rand(t, heads, generator=g)
    wide = _columns(gate, 8)
    z, od = gate.double(), o.double().view(t, heads, dim)
    tol = 3e-6 if dtype == torch.float32 else 4e-3

    def run(**kw):
        out = torch.empty(t, n, dtype=dtype, device=DEV)
        ops.gated_rmsnorm(o.to(DEV), wide, w.to(DEV), eps, out, **kw)
        return out
    first = (od.reshape(t, n) * plain.silu(z)).view(t, heads, dim)
    assert rel_err(run(group=dim, gate_act="silu", gate_first=True),
                   plain.unit(first, eps).reshape(t, n) * w.double()) < tol
    assert rel_err(run(gate_act="silu", gate_first=True), plain.unit(first.reshape(t, n), eps) * w.double()) < tol
    assert rel_err(run(group=dim, den=den.to(DEV)),
                   plain.unit(od / den.double()[:, :, None], eps).reshape(t, n) * w.double() * torch.sigmoid(z)) < tol


@pytest.mark.parametrize("rows", [1, 7, 16, 29])
def test_two_few_row_products_together(ops, rows):
    """A narrow product wanted in 32-bit beside a wide one of the same rows, in either order, and
    two products of different rows and widths: what they give held back and launched together is
    what they give by themselves."""
    g = torch.Generator().manual_seed(rows)
    k = 256
    x, y = (torch.randn(rows, n, generator=g).to(torch.bfloat16).to(DEV) for n in (k, 2 * k))
    w = [(torch.randn(n, m, generator=g) * 0.1).to(torch.bfloat16).to(DEV) for n, m in ((10, k), (712, k), (96, k), (96, 2 * k))]
    pairs = [((x, w[0], torch.float32), (x, w[1], torch.bfloat16)), ((x, w[1], torch.bfloat16), (x, w[0], torch.float32)),
             ((x, w[2], torch.bfloat16), (y, w[3], torch.bfloat16))]
    for pair in pairs:
        outs = [torch.full((rows, m.shape[0]), float("nan"), dtype=d, device=DEV) for _, m, d in pair]
        with ops.together():
            for (a, m, _), out in zip(pair, outs):
                ops.linear(a, m, out)
        for (a, m, d), out in zip(pair, outs):
            assert rel_err(out, a.double().cpu() @ m.double().cpu().T) < (1e-6 if d == torch.float32 else 4e-3)


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


def _rows(tables, who):
    width = max(len(t) for t in tables)
    return torch.tensor([tables[r] + [-1] * (width - len(tables[r])) for r in who], dtype=torch.int32, device=DEV)


@pytest.mark.parametrize("dtype,plain_kernel", KERNELS, indirect=["plain_kernel"])
@pytest.mark.parametrize("heads,kv,dim,vdim,rot,rows", [
    (6, 3, 20, 12, 10, 1), (4, 2, 64, 64, 64, 1), (8, 2, 64, 32, 32, 1), (2, 1, 88, 72, 40, 1), (2, 2, 16, 16, 0, 1),
    (1, 1, 8, 40, 8, 1), (16, 4, 128, 128, 64, 16), (4, 1, 96, 48, 32, 16), (40, 8, 256, 256, 32, 16)])
def test_unit_heads_on_their_way_to_attention(ops, dtype, plain_kernel, heads, kv, dim, vdim, rot, rows):
    """Rotation at frequencies divided by a factor, every query and key head divided by its root
    mean square, the cache write: three requests in portions and single rows."""
    from ninfer_amd.parts import Rotary
    g = torch.Generator().manual_seed(dim + heads)
    lens, ps, eps = [45 * rows, 7, 30 * rows], 8, 1e-3
    nq, nk, nv = heads * dim, kv * dim, kv * vdim
    ch = nq + nk + nv
    u_all = [(torch.randn(n, ch, generator=g) * torch.rand(n, 1, generator=g) * 0.3).to(dtype) for n in lens]
    r = {"base": 300.0, "dims": rot, "scaling": {"factor": 2.5}}
    freq = Rotary(rot, 300.0, scaling={"factor": 2.5}).inv_freq() if rot else None
    tables, pages = _tables([-(-n // ps) for n in lens], 2, g)
    k_pool = torch.full((pages, kv, ps, dim), float("nan"), dtype=dtype, device=DEV)
    v_pool = torch.full((pages, kv, ps, vdim), float("nan"), dtype=dtype, device=DEV)
    got_q = [torch.zeros(n, nq) for n in lens]
    cuts = [_cut(lens[0], [13, 2, (9 if rows == 1 else 36 * rows + 1), 3], 6), _cut(7, [3, 2], 2),
            _cut(lens[2], [2, 11 * rows, 1, 8], 4)]
    for ctx, who, starts, counts in _steps(ops, dtype, cuts, [0, 1, 2]):
        u = _columns(torch.cat([u_all[i][s:s + n] for i, s, n in zip(who, starts, counts)]), 8)
        q = torch.empty(ctx.T, nq, dtype=dtype, device=DEV)
        ops.qkv_wide(u, ctx, q, heads, kv, dim, vdim, k_pool, v_pool, _rows(tables, who), ps, norm_eps=eps,
                     inv_freq=freq.to(DEV) if rot else None, rot_dim=rot, unit_heads=True)
        o = 0
        for i, s, n in zip(who, starts, counts):
            got_q[i][s:s + n] = q[o:o + n].float().cpu()
            o += n
    tol = (3e-6 if rows == 1 else 1e-5) if dtype == torch.float32 else 6e-3
    for i, n in enumerate(lens):
        x, pos = u_all[i].double(), torch.arange(n)
        q = plain.unit(plain.rotate(x[:, :nq].reshape(n, heads, dim), pos, r), eps)
        k = plain.unit(plain.rotate(x[:, nq:nq + nk].reshape(n, kv, dim), pos, r), eps)
        table = torch.tensor(tables[i])
        assert rel_err(got_q[i], q.reshape(n, -1)) < tol
        assert rel_err(_gather(k_pool.cpu(), table, n, ps), k) < tol
        assert torch.equal(_gather(v_pool.cpu(), table, n, ps), u_all[i][:, nq + nk:].reshape(n, kv, vdim))


SHAPES = [(6, 3, 20, 12, 4), (8, 2, 64, 32, 16), (4, 4, 32, 96, 8), (6, 2, 88, 72, 16), (3, 1, 128, 128, 32), (2, 2, 8, 24, 8),
          (40, 1, 16, 16, 4), (16, 4, 64, 64, 16), (8, 2, 128, 128, 16), (6, 1, 128, 128, 64), (5, 1, 96, 96, 16)]


@pytest.mark.parametrize("dtype,plain_kernel", KERNELS, indirect=["plain_kernel"])
@pytest.mark.parametrize("gated", [True, False])
@pytest.mark.parametrize("heads,kv,dim,vdim,ps", SHAPES)
def test_attention_with_learned_sinks(ops, dtype, plain_kernel, gated, heads, kv, dim, vdim, ps):
    """Three requests: whole prompts in one step, then a step that mixes single rows with a
    portion, then single rows alone, against the plain softmax. The heads' sinks range from
    next to nothing to far above every score, so that a sink left out, counted twice, scaled or
    taken from another head shows."""
    g = torch.Generator().manual_seed(heads * dim + 1)
    lens, scale = [310, 37, 141], 0.9 / math.sqrt(dim)
    ks = [torch.randn(n, kv, dim, generator=g).to(dtype) for n in lens]
    vs = [torch.randn(n, kv, vdim, generator=g).to(dtype) for n in lens]
    qs = [torch.randn(n, heads, dim, generator=g).to(dtype) for n in lens]
    gates = [torch.randn(n, heads * vdim, generator=g).to(dtype) for n in lens]
    sinks = torch.linspace(-30.0, 9.0, heads) if heads > 1 else torch.tensor([2.5])
    sinks = sinks[torch.randperm(heads, generator=g)]
    tables, pages = _tables([-(-n // ps) for n in lens], 3, g)

    def lay(rows):
        pool = torch.full((pages, kv, ps, rows[0].shape[2]), float("nan"), dtype=dtype)
        for r, x in enumerate(rows):
            js = torch.arange(x.shape[0])
            pool[torch.tensor(tables[r])[js // ps], :, js % ps] = x
        return pool.to(DEV)
    k_pool, v_pool = lay(ks), lay(vs)
    want = []
    for r in range(3):
        o = plain.attend(qs[r].double(), ks[r].double(), vs[r].double(), scale, sinks).reshape(lens[r], -1)
        want.append(o * torch.sigmoid(gates[r].double()) if gated else o)
    tol = 2e-5 if dtype == torch.float32 else 1.2e-2
    for step in ([(0, 0, 310), (1, 0, 37), (2, 0, 141)], [(1, 36, 1), (2, 69, 1), (0, 97, 213)],
                 [(0, 309, 1), (1, 20, 1), (2, 64, 1)], [(2, 3, 2), (0, 60, 33)], [(0, 200, 1)], [(2, 0, 1)]):
        ctx = util.make_context(ops, dtype, [(s, n) for _, s, n in step])
        ctx.single_rows = sum(1 for _, _, n in step if n == 1) if step[0][2] == 1 else 0
        rows = torch.cat([qs[r][s:s + n] for r, s, n in step]).reshape(ctx.T, heads * dim).to(DEV)
        gate = _columns(torch.cat([gates[r][s:s + n] for r, s, n in step]), 8) if gated else None
        out = torch.full((ctx.T, heads * vdim), float("nan"), dtype=dtype, device=DEV)
        ops.paged_attention(rows, k_pool, v_pool, _rows(tables, [r for r, _, _ in step]), ctx, heads, kv, dim, ps, None,
                            scale, out, vdim=vdim, sink=True, sinks=sinks.to(DEV), gate=gate)
        ref = torch.cat([want[r][s:s + n] for r, s, n in step]).reshape(ctx.T, heads, vdim)
        got = out.view(ctx.T, heads, vdim)
        assert torch.isfinite(out).all()
        for h in range(heads):    # (a head behind a loud sink is small beside the others)
            assert rel_err(got[:, h], ref[:, h]) < tol, (step, h, float(sinks[h]))


@pytest.mark.parametrize("dtype,plain_kernel", KERNELS, indirect=["plain_kernel"])
@pytest.mark.parametrize("dim,vdim,ps", [(32, 32, 8), (96, 40, 16), (128, 128, 16)])
def test_one_loud_key_anywhere_before_a_sink(ops, dtype, plain_kernel, dim, vdim, ps):
    """Among hundreds of keys that score 0 one that stands out, with a value no other has: the
    request's first, at both sides of pages' and tiles' borders, the row's own, and the one after
    it, which is not seen; for rows inside prompt portions and for decoded ones. A sink as loud as
    the key halves what is seen of it."""
    n, heads = 330, 4
    rows_at = [0, 1, 63, 64, 127, 128, 200, 329]
    g = torch.Generator().manual_seed(dim)
    tables, pages = _tables([-(-n // ps)], 2, g)
    js = torch.arange(n)
    sinks = torch.tensor([-40.0, 12.0, -40.0, 12.0])
    q = torch.zeros(n, heads, dim)
    q[:, :, 0] = 1.0
    for loud in (0, 1, ps - 1, ps, 63, 64, 127, 128, 200, 201):
        k, v = torch.zeros(n, 2, dim), torch.zeros(n, 2, vdim)
        k[loud, :, 0] = 12.0
        v[loud] = 8.0
        pools = []
        for x in (k, v):
            pool = torch.full((pages, 2, ps, x.shape[2]), float("nan"), dtype=dtype)
            pool[torch.tensor(tables[0])[js // ps], :, js % ps] = x.to(dtype)
            pools.append(pool.to(DEV))
        want = plain.attend(q.double(), k.double(), v.double(), 1.0, sinks)
        assert want[loud, 0, 0] > 7.9 and abs(want[loud, 1, 0] - 4.0) < 0.1 and (loud == 0 or want[loud - 1, 0, 0] == 0)
        for first, count in [(0, n), (150, 60)] + [(r, 1) for r in rows_at]:
            ctx = util.make_context(ops, dtype, [(first, count)])
            ctx.single_rows = 1 if count == 1 else 0
            out = torch.full((count, heads * vdim), float("nan"), dtype=dtype, device=DEV)
            ops.paged_attention(q[first:first + count].reshape(count, -1).to(dtype).to(DEV), pools[0], pools[1],
                                _rows(tables, [0]), ctx, heads, 2, dim, ps, None, 1.0, out, vdim=vdim, sink=True,
                                sinks=sinks.to(DEV))
            diff = (out.double().cpu().view(count, heads, vdim) - want[first:first + count]).abs().max()
            assert diff < (1e-4 if dtype == torch.float32 else 0.05), (loud, first, count)


def _scan_requests(lens):
    """Cuts and slots for three requests whose state lies in a wider tensor's rows."""
    cuts = []
    for i, n in enumerate(lens):
        sizes = [[2, 129, 3, 40], [5, 2], [n]][i % 3]
        cuts.append(_cut(n, sizes, min(3, n - 2) if n > 2 else 0))
    return cuts, [3, 0, 4][:len(lens)]


SCANS = [[45, 7, 30], [400, 9, 130], [128, 256, 20], [700, 2, 2]]


@pytest.mark.parametrize("dtype,plain_kernel", KERNELS, indirect=["plain_kernel"])
@pytest.mark.parametrize("lens", SCANS)
@pytest.mark.parametrize("heads,groups,dim,vdim", [(6, 3, 12, 10), (4, 2, 64, 32), (3, 1, 33, 7), (2, 1, 128, 72), (4, 4, 8, 8),
                                                   (1, 1, 256, 64), (2, 2, 400, 16), (5, 1, 40, 136)])
def test_state_space_scan(ops, dtype, plain_kernel, lens, heads, groups, dim, vdim):
    """The recurrence with a step size per head and token: portions (row by row, and in chunks of
    the matrix cores), single rows beside them and alone, states in slots of a wider tensor. The
    rates range from all but no decay to nothing left a row later."""
    g = torch.Generator().manual_seed(dim + vdim + lens[0])
    inner, gn = heads * vdim, groups * dim
    xs = [torch.randn(n, inner + 2 * gn, generator=g).to(dtype) for n in lens]
    zs = [torch.randn(n, heads, generator=g) * 2 for n in lens]
    bias, rate = torch.randn(heads, generator=g) - 2, torch.logspace(-3, 1.5, heads)
    skip = torch.randn(heads, generator=g)
    floats = heads * dim * vdim
    state = torch.zeros(5, floats + 8, device=DEV)
    got = [torch.zeros(n, inner) for n in lens]
    cuts, slots = _scan_requests(lens)
    for ctx, who, starts, counts in _steps(ops, dtype, cuts, slots):
        pick = lambda t: torch.cat([t[r][s:s + n] for r, s, n in zip(who, starts, counts)])
        out = torch.full((ctx.T, inner), float("nan"), device=DEV)
        ops.state_space(pick(xs).to(DEV), heads, vdim, dim, groups, pick(zs).to(DEV), bias.to(DEV), rate.to(DEV),
                        skip.to(DEV), state[:, 4:-4], ctx, out)
        o = 0
        for r, s, n in zip(who, starts, counts):
            got[r][s:s + n] = out[o:o + n].cpu()
            o += n
    for r, n in enumerate(lens):
        x = xs[r].double()
        dt = plain.softplus(zs[r].double() + bias.double())
        v, b, c = x[:, :inner].view(n, heads, vdim), x[:, inner:inner + gn].view(n, groups, dim), x[:, inner + gn:].view(n, groups, dim)
        y, last = plain.state_space(v, b, c, dt, rate.double())
        y = y + skip.double()[:, None] * v
        have = got[r].view(n, heads, vdim)
        for h in range(heads):
            assert rel_err(have[:, h], y[:, h]) < 2e-5, (r, h)
        assert rel_err(state[slots[r], 4:4 + floats], last.reshape(-1)) < 2e-5
    assert (state[:, :4] == 0).all() and (state[:, -4:] == 0).all() and (state[1:3] == 0).all()


@pytest.mark.parametrize("dtype,plain_kernel", KERNELS, indirect=["plain_kernel"])
@pytest.mark.parametrize("lens", SCANS)
@pytest.mark.parametrize("heads,dim,vdim,cap", [(3, 14, 9, 6.0), (4, 32, 64, 12.0), (5, 6, 11, 20.0), (2, 128, 72, 15.0),
                                                (1, 8, 8, 3.0), (2, 256, 128, 10.0), (1, 72, 300, 12.0)])
def test_matrix_memory(ops, dtype, plain_kernel, lens, heads, dim, vdim, cap):
    """Exponential gates with a running maximum, the divisor, the head norm and the output gate,
    in the same cuts. Gates wide enough that the running maximum follows the write gate in some
    rows and the forget gate in others, that the divisor is the product with the keys' sum in
    some and e^(-m) in others, and a start at m = 0 counts (the first write gates lie below it)."""
    g = torch.Generator().manual_seed(dim + vdim + lens[0])
    qk, nv, eps = heads * dim, heads * vdim, 1e-6
    us = [torch.randn(n, 2 * qk + 2 * nv, generator=g).to(dtype) for n in lens]
    zs = [torch.randn(n, 2 * heads, generator=g) * 4 for n in lens]
    for z in zs:
        z[:3, :heads] -= 6.0
    bias = torch.cat([torch.randn(heads, generator=g), torch.linspace(-2, 6, heads)])
    norm_w = 1 + 0.3 * torch.randn(nv, generator=g)
    floats = heads * (dim * vdim + dim + 1)
    room = -(-floats // 4) * 4
    state = torch.zeros(5, room + 8, device=DEV)
    got = [torch.zeros(n, nv) for n in lens]
    cuts, slots = _scan_requests(lens)
    for ctx, who, starts, counts in _steps(ops, dtype, cuts, slots):
        pick = lambda t: torch.cat([t[r][s:s + n] for r, s, n in zip(who, starts, counts)])
        u = _columns(pick(us), 8)
        out = torch.full((ctx.T, nv), float("nan"), dtype=dtype, device=DEV)
        ops.matrix_memory(u, 0, qk, 2 * qk, pick(zs).to(DEV), bias.to(DEV), heads, dim, vdim, cap, dim ** -0.5,
                          state[:, 4:-4], ctx, u[:, 2 * qk + nv:], norm_w.to(DEV), eps, out)
        o = 0
        for r, s, n in zip(who, starts, counts):
            got[r][s:s + n] = out[o:o + n].float().cpu()
            o += n
    tol = 3e-5 if dtype == torch.float32 else 4e-3
    for r, n in enumerate(lens):
        u = us[r].double()
        z = plain.capped(zs[r].double() + bias.double(), cap)
        write, keep = z[:, :heads], plain.log_sigmoid(z[:, heads:])
        q = u[:, :qk].view(n, heads, dim) * dim ** -0.5
        k, v = u[:, qk:2 * qk].view(n, heads, dim), u[:, 2 * qk:2 * qk + nv].view(n, heads, vdim)
        o, (S, nn, m) = plain.memory(q, k, v, write, keep)
        want = plain.unit(o, eps).reshape(n, nv) * norm_w.double() * torch.sigmoid(u[:, 2 * qk + nv:])
        have, want = got[r].view(n, heads, vdim), want.view(n, heads, vdim)
        for h in range(heads):
            assert rel_err(have[:, h], want[:, h]) < tol, (r, h)
        st = state[slots[r], 4:4 + floats].cpu().double()
        assert rel_err(st[:qk * vdim], S.reshape(-1)) < 1e-4 and rel_err(st[qk * vdim:qk * (vdim + 1)], nn.reshape(-1)) < 1e-4
        assert (st[qk * (vdim + 1):] - m).abs().max() < 1e-3
    assert (state[:, :4] == 0).all() and (state[:, -4:] == 0).all() and (state[1:3] == 0).all()


@pytest.mark.parametrize("dtype", BOTH)
def test_states_remember_and_forget(ops, dtype):
    """A loud token hundreds of rows back, in a prompt of one piece, in portions across chunk
    borders and token by token: a head that does not decay has it to the end, one that decays
    at once has nothing of it a row later."""
    n, dim, vdim = 600, 8, 16
    x = torch.zeros(n, 2 * vdim + 2 * dim)
    x[:, 2 * vdim + dim:] = 1.0                    # C
    x[3, 2 * vdim:2 * vdim + dim] = 1.0            # B of row 3 alone
    x[3, :2 * vdim] = 100.0
    x = x.to(dtype)
    z, rate = torch.full((n, 2), 1.0), torch.tensor([1e-6, 60.0])
    dt = plain.softplus(z.double())
    v = x[:, :2 * vdim].double().view(n, 2, vdim)
    want, _ = plain.state_space(v, x[:, 2 * vdim:2 * vdim + dim].double().view(n, 1, dim),
                                x[:, 2 * vdim + dim:].double().view(n, 1, dim), dt, rate.double())
    assert want[-1, 0, 0] > 900 and abs(want[4, 1, 0]) < 1e-20
    zero = torch.zeros(2, device=DEV)
    for cut in ([n], [257, 2, 341], [128, 128, 344], _cut(n, [590], 10)):
        state, got = torch.zeros(1, 2 * dim * vdim, device=DEV), []
        for ctx, _, starts, counts in _steps(ops, dtype, [cut], [0]):
            s, c = starts[0], counts[0]
            out = torch.empty(ctx.T, 2 * vdim, device=DEV)
            ops.state_space(x[s:s + c].to(DEV), 2, vdim, dim, 1, z[s:s + c].to(DEV), zero, rate.to(DEV), zero, state, ctx, out)
            got.append(out.cpu())
        got = torch.cat(got).view(n, 2, vdim).double()
        # (a decay this close to 1 is rounded alike in every row)
        assert (got - want).abs().max() < 1e-4 * want.abs().max()


@pytest.mark.parametrize("dtype", BOTH)
def test_memory_keeps_a_loud_row_and_its_maximum(ops, dtype):
    """The same for the matrix memory: one row writes loudly, hundreds of quiet ones follow, and a
    head that does not forget hands its value back to the end, one that forgets at once does not.
    The running maximum falls with the forget gate alone, in the state too."""
    n, heads, dim, vdim, cap = 500, 2, 8, 16, 15.0
    u = torch.zeros(n, 2 * heads * dim + 2 * heads * vdim)
    u[:, :2 * heads * dim] = 1.0
    v0 = 2 * heads * dim
    u[:, v0:v0 + heads * vdim] = 0.01 * torch.randn(n, heads * vdim, generator=torch.Generator().manual_seed(2))
    u[5, v0:v0 + heads * vdim] = torch.arange(heads * vdim) - 10.0
    u = u.to(dtype)
    z = torch.tensor([-9.0, -9.0, 60.0, -7.0]).repeat(n, 1)     # write gates, then forget gates
    z[5, :2] = 8.0
    zc = plain.capped(z.double(), cap)
    q = u[:, :heads * dim].double().view(n, heads, dim) * dim ** -0.5
    k, v = u[:, heads * dim:v0].double().view(n, heads, dim), u[:, v0:v0 + heads * vdim].double().view(n, heads, vdim)
    o, (S, nn, m) = plain.memory(q, k, v, zc[:, :2], plain.log_sigmoid(zc[:, 2:]))
    want = plain.unit(o, 1e-6)
    loud = plain.unit(v[5], 1e-6)
    assert rel_err(want[-1, 0], loud[0]) < 1e-2 and rel_err(want[-1, 1], loud[1]) > 0.5
    zero, one = torch.zeros(2 * heads, device=DEV), torch.ones(heads * vdim, device=DEV)
    for cut in ([n], [130, 2, 368], [128, 128, 244], _cut(n, [490], 10)):
        state, got = torch.zeros(1, heads * (dim * vdim + dim + 1) + 2, device=DEV), []
        for ctx, _, starts, counts in _steps(ops, dtype, [cut], [0]):
            s, c = starts[0], counts[0]
            part = u[s:s + c].to(DEV)
            out = torch.empty(ctx.T, heads * vdim, dtype=dtype, device=DEV)
            ops.matrix_memory(part, 0, heads * dim, v0, z[s:s + c].to(DEV), zero, heads, dim, vdim, cap, dim ** -0.5, state,
                              ctx, part[:, v0 + heads * vdim:], one, 1e-6, out)
            got.append(2 * out.float().cpu())       # (the gate's logits are 0: a factor of 1 / 2)
        got = torch.cat(got).view(n, heads, vdim)
        assert rel_err(got, want) < (1e-4 if dtype == torch.float32 else 5e-3), cut
        assert (state[0, heads * dim * (vdim + 1):heads * dim * (vdim + 1) + heads].double().cpu() - m).abs().max() < 1e-3


# ---- whole models ----------------------------------------------------------------------------

PROMPT_LENGTHS = [70, 1, 23, 97, 40, 64]


def row_errors(got, ref):
    d = (got - ref).double()
    return (d - d.mean(-1, keepdim=True)).pow(2).mean(-1).sqrt() / ref.double().std()


def noise_of(cfg, w, toks, ref):
    """How far the plain implementation's logits move when every weight is disturbed by one
    part in 2^9 (what rounding to bfloat16 does to a number), several times for short requests:
    median, ninth decile and largest of the rows' errors. The comparisons' bounds come from
    the model at hand."""
    g = torch.Generator().manual_seed(len(toks))
    errs = []
    for _ in range(6 if len(toks) <= 100 else 2):
        w2 = {k: v * (1 + torch.randn(v.shape, generator=g) * 2.0 ** -9) for k, v in w.items()}
        errs.append(row_errors(plain.forward(cfg, w2, toks)[0], ref))
    mid = torch.stack(errs).mean(0)
    return mid.median().item(), mid.kthvalue(max(1, int(0.9 * len(mid)))).values.item(), \
        torch.stack(errs).max().item()


@pytest.fixture(scope="module", params=list(nosedra_cases.CASES))
def case(request, tmp_path_factory):
    import ninfer_amd
    name = request.param
    make, seed = nosedra_cases.CASES[name]
    raw = make()
    out = {"name": name, "cfg": raw, "dirs": {}, "ref": {}, "noise": {},
           "reqs": {f"r{i}": util.random_tokens(n, raw["vocab"], 50 + i) for i, n in enumerate(PROMPT_LENGTHS)}}
    for dtype in ("float32", "bfloat16"):
        d = str(tmp_path_factory.mktemp(f"nosedra_{name}_{dtype}"))
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
        f50, f90, fmax, floor = (3, 4, 3, 0.03) if dtype == "bfloat16" else \
            (8 * 2.0 ** -15, 8 * 2.0 ** -15, 16 * 2.0 ** -15, 3e-6)
        e50 = err.median().item()
        e90 = err.kthvalue(max(1, int(0.9 * len(err)))).values.item()
        if len(err) >= 20:
            assert e50 <= max(f50 * n50, floor), f"{who}: median row error {e50:.2e} (disturbance {n50:.2e})"
            assert e90 <= max(f90 * n90, floor), f"{who}: ninth decile {e90:.2e} (disturbance {n90:.2e})"
        assert err.max().item() <= max(fmax * nmax, 4 * floor), \
            f"{who}: row {err.argmax()} is off by {err.max():.2e} (disturbance {nmax:.2e})"


def test_layer_by_layer(case):
    """The 32-bit residual stream after every layer, for a prompt in one step and in portions;
    bounds from how far the plain streams move when every weight is off by 32-bit rounding (a
    head whose output all but cancels in front of its norm carries that far)."""
    from ninfer_amd.engine import Chunk
    cfg, w = util.read_folder(case["dirs"]["float32"])
    toks = case["reqs"]["r4"]
    streams = plain.forward(cfg, w, toks)[1]
    g = torch.Generator().manual_seed(1)
    off = {k: v.double() * (1 + torch.randn(v.shape, generator=g, dtype=D) * 2.0 ** -24) for k, v in w.items()}
    moved = [rel_err(a, b) for a, b in zip(plain.forward(cfg, off, toks)[1], streams)]
    runner = make_runner(case, "float32")
    assert len(runner.spec.plan) == len(streams)
    got = []

    def tap(i, residual, pending):
        whole = residual.clone()
        runner.ops.stream_norm(whole, pending)     # (what the layer leaves to the next one's norm)
        got[i].append(whole.cpu())
    for cuts in ([len(toks)], [17, 2, len(toks) - 19]):
        slot = runner.open()
        got[:] = [[] for _ in streams]
        runner.tap = tap
        o = 0
        for n in cuts:
            runner.step([Chunk(slot, toks[o:o + n], [])])
            o += n
        runner.tap = None
        runner.close(slot)
        for i, want in enumerate(streams):
            g = torch.cat(got[i]).double()
            assert rel_err(g, want) < max(2e-6, 8 * moved[i]), f"layer {i}"


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
    runner = make_runner(case, dtype, page_size=8, num_pages=38)
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
    recurrent state and convolution inputs still in it unless it is cleared."""
    runner = make_runner(case, "float32", seqs=1)
    for rid in ("r3", "r0", "r1", "r2"):
        toks = case["reqs"][rid]
        sched = util.schedule_tail(rid, toks, 5) if len(toks) > 1 else util.schedule_whole(rid, toks)
        check_logits(case, "float32", util.run_schedule(runner, sched), "slot used again")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_decoding(case, dtype):
    """A few tokens of prompt, then hundreds of single steps: across pages and the attention
    kernels' tiles, with the recurrent states carried on."""
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
    several chunks of the recurrences among them."""
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
    the plain implementation."""
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


@pytest.mark.parametrize("seed", ["state-space layers alone", "parallel layers alone"] + list(range(10)))
def test_random_configurations(seed, tmp_path):
    """Configurations drawn at random (sizes, head counts, kinds and order of layers, what is
    absent), and models of one kind of layer, in both precisions: whole, in portions and in a
    mixed batch."""
    import ninfer_amd
    from ninfer_amd import EngineOptions, load_model
    raw = nosedra_cases.alone(seed.split()[0]) if isinstance(seed, str) else nosedra_cases.random_config(seed)
    seed = len(seed) if isinstance(seed, str) else seed
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
    assert all(g["in_use"] == 0 for g in stats["groups"])
    prompt = case["reqs"]["r2"][:9]
    p = subprocess.run([sys.executable, os.path.join(root, "bin", "ninfer"), case["dirs"]["float32"], "--dtype",
                        "float32", "--prompt-ids", ",".join(map(str, prompt)), "--max-new", "4", "--temperature",
                        "0", "--max-context", "64"], text=True, capture_output=True, timeout=600)
    assert p.returncode == 0, p.stderr[-2000:]
    cfg, w = util.read_folder(case["dirs"]["float32"])
    first = int(plain.forward(cfg, w, prompt)[0][-1].argmax())
    assert str(first) in p.stdout
