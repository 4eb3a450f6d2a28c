"""Rudazen without a GPU: the configuration reader, the model the builder makes (tensor names
and shapes, caches, state), the cache manager's groups of blocks, the plain implementation's
own properties (which blocks are seen, means, frequencies with their ramp, the recurrence in
pieces), and the engine's host logic on plain stand-ins for the kernels."""
import copy
import math

import pytest
import torch

import plain_rudazen as plain
import rudazen_cases
import util

D = torch.float64
STD = 0.25


def _spec(raw):
    from ninfer_amd import build_spec
    return build_spec(raw)


# ---- reader and builder ----------------------------------------------------------------------

def test_reader_reads_every_key():
    cfg, _ = _spec(rudazen_cases.config_odd())
    assert (cfg.vocab, cfg.width, cfg.eps, cfg.alpha, cfg.embedding_scale) == (211, 72, 1e-5, 1.7, 5.5)
    a = cfg.layers[0].mixer
    assert (a.heads, a.kv_heads, a.dim, a.vdim, a.window, a.pool) == (6, 3, 20, 20, 11, 3)
    assert (a.rot.dims, a.rot.base, a.rot.scaling) == (10, 500.0, None) and a.scale == 1 / math.sqrt(20)
    m = cfg.layers[1].mixer
    assert (m.left.heads, m.left.kv_heads, m.left.dim, m.left.vdim, m.left.window, m.left.pool) == (6, 2, 12, 20, 17, None)
    s = m.left.rot.scaling
    assert (s.factor, s.original, s.fast, s.slow) == (3.0, 24, 4.0, 0.5)
    assert (m.right.heads, m.right.dim, m.right.vdim) == (3, 12, 20)
    assert [x.ff for x in cfg.layers] == [40, 56, None, 24]
    ones, _ = _spec(rudazen_cases.config_ones())
    assert ones.layers[1].mixer.window is None and ones.layers[3].mixer.pool is None
    assert ones.layers[0].mixer.pool == 1 and ones.layers[2].mixer.left.rot.dims == 0


@pytest.mark.parametrize("change,word", [
    (lambda c: c.pop("vocab"), "vocab"),
    (lambda c: c.pop("postln_alpha"), "postln_alpha"),
    (lambda c: c["norm"].pop("eps"), "eps"),
    (lambda c: c["layers"][0].update(type="linear"), "type"),
    (lambda c: c["layers"][0]["mixer"].update(heads=5), "heads"),
    (lambda c: c["layers"][0]["mixer"].update(vdim=16), "vdim"),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=7), "rot.dims"),
    (lambda c: c["layers"][0]["mixer"]["mask"].update(pool=0), "pool"),
    (lambda c: c["layers"][0]["mixer"]["mask"].pop("size"), "mask.pool"),
    (lambda c: c["layers"][1]["mixer"]["left"]["mask"].update(pool=4), "mask.pool"),
    (lambda c: c["layers"][1]["mixer"]["left"]["rot"]["scaling"].update(fast=0.0), "scaling"),
    (lambda c: c["layers"][1]["mixer"].pop("right"), "right"),
    (lambda c: c["layers"][1]["mlp"].update(kind="moe"), "kind"),
    (lambda c: c["layers"][0]["mixer"].update(scale=-1.0), "scale"),
])
def test_reader_names_the_key_it_refuses(change, word):
    from ninfer_amd.config import ConfigError
    raw = copy.deepcopy(rudazen_cases.config_odd())
    change(raw)
    with pytest.raises(ConfigError, match=word):
        _spec(raw)


@pytest.mark.parametrize("name", list(rudazen_cases.CASES))
def test_builder_names_every_tensor(name):
    raw = rudazen_cases.CASES[name][0]()
    _, spec = _spec(raw)
    specs = {k: v.shape for k, v in spec.tensor_specs().items()}
    w = raw["width"]
    want = {"embed": (raw["vocab"], w), "head": (raw["vocab"], w), "final.norm": (w,)}
    for i, layer in enumerate(raw["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        want[p + "norm1"] = (w,)

        def heads(q, m, values):
            nq, nk = m["heads"] * m["dim"], m["kv_heads"] * m["dim"]
            want.update({q + "q": (nq, w), q + "k": (nk, w), q + "q.norm": (nq,), q + "k.norm": (nk,),
                         q + "o": (w, m["heads"] * m["vdim"])})
            if values:
                want[q + "v"] = (m["kv_heads"] * m["vdim"], w)
        if layer["type"] == "attention":
            heads(p + "mix.", m, False)
        else:
            left, right = m["left"], m["right"]
            heads(p + "mix.left.", left, True)
            want[p + "mix.left.temp"] = (left["heads"],)
            want[p + "mix.left.g"] = (left["heads"] * left["vdim"], w)
            qk, v, q = right["heads"] * right["dim"], right["heads"] * right["vdim"], p + "mix.right."
            want.update({q + "q": (qk, w), q + "f": (qk, w), q + "f.b": (qk,), q + "lower": (qk,), q + "v": (v, w),
                         q + "norm": (right["vdim"],), q + "o": (w, v), q + "out": (w,), p + "mix.left.out": (w,)})
        if layer["mlp"]:
            ff = layer["mlp"]["ff"]
            want.update({p + "norm2": (w,), p + "mlp.gate": (ff, w), p + "mlp.up": (ff, w), p + "mlp.down": (w, ff)})
    assert specs == want


def test_caches_and_state():
    """A layer with blocks keeps its window (or a whole block, when that is longer) per token
    and a mean per block of all positions; two mixers side by side keep the left one's window
    and the right one's state; layers of equal kind share page numbers."""
    _, spec = _spec(rudazen_cases.config_odd())
    mixers = [b.mixer for b in spec.blocks]
    need = mixers[0].cache_need()
    assert (need.window, need.stride, need.blocks.window, need.blocks.stride) == (11, 1, None, 3)
    assert [(p.name, p.outer, p.inner) for p in need.all_needs()[1].pools] == \
        [("k_block", (3,), (20,)), ("v_block", (3,), (20,))]
    assert mixers[2].cache_need().window == 7 and mixers[2].window == 5     # a block is longer than the window
    assert mixers[1].cache_need().window == 17 and mixers[1].cache_need().blocks is None
    assert mixers[1].state_floats() == 3 * 12 * 20 and mixers[0].state_floats() == 0
    assert need.bytes_per_token(2) == 2 * 3 * 20 * 2 + -(-2 * 3 * 20 * 2 // 3)


def test_forget_gates_bounds_are_checked():
    from ninfer_amd.parts import ForgetGateAttention, WeightBinder
    part = ForgetGateAttention("m.", 8, 1, 4, 4, 1e-5)
    w = util.random_part_weights(part, 1)
    assert ((w["m.lower"] > 0) & (w["m.lower"] < 1)).all()
    w["m.lower"][2] = 1.25
    with pytest.raises(ValueError, match="lower"):
        part.bind_all(WeightBinder(util.DictSource(w), torch.device("cpu"), torch.float32))


def test_parameters_that_do_not_go_together_are_refused():
    from ninfer_amd.parts import Attention, NoPosition, Rotary
    base = dict(prefix="a.", hidden=16, heads=2, kv_heads=1, head_dim=8, position=NoPosition(), qkv_bias=False)
    for more in (dict(values="keys", vdim=4), dict(pool=4), dict(pool=2, window=4, conv_taps=2),
                 dict(output_gate=True, qk_norm_eps=1e-5), dict(qk_norm="rows"),
                 dict(position=Rotary(8, 100.0, scaling=dict(factor=2.0, original=8, fast=4.0, slow=1.0)),
                      qkv_bias=True)):
        with pytest.raises(ValueError):
            Attention(**{**base, **more})


# ---- the cache manager's groups of blocks ----------------------------------------------------

def _need(window, block):
    from ninfer_amd.parts import CacheNeed
    return CacheNeed.keys_values(1, 4, window, block=block)


def test_pages_of_blocks_are_taken_as_blocks_become_whole():
    from ninfer_amd.cache.manager import CacheManager
    m = CacheManager([_need(6, 3), _need(6, 3), _need(9, None)], 4, 20, 2, 64)
    assert [(g.window, g.stride, g.max_pages) for g in m.groups] == [(6, 1, 16), (None, 3, 6), (9, 1, 16)]
    assert m.groups[1].instances == [0, 1] and m.block_group_of_instance == {0: 1, 1: 1}
    assert m.groups[1].allocator.num_pages == 9       # 80 tokens: 7 pages of 4 blocks, and one each for 2 requests
    m.allocate_pools("cpu", torch.float32)
    assert sorted(m.pools[0]) == ["k", "k_block", "v", "v_block"] and sorted(m.pools[2]) == ["k", "v"]
    assert m.pools[0]["k_block"].shape == (9, 1, 4, 4)
    s = m.acquire()
    for n, pages in ((2, 0), (3, 1), (14, 1), (15, 2), (26, 2), (27, 3)):
        m.reserve(s, n)
        m.commit(s, n)
        assert len(m.groups[1].tables[s]) == pages, n
    assert m.groups[0].window_freed == 5 and all(p >= 0 for p in m.groups[1].tables[s])
    m.check()
    m.release(s)
    assert all(g.allocator.in_use == 0 for g in m.groups)


def test_freed_pages_of_blocks_are_poisoned_in_their_own_pools():
    from ninfer_amd.cache.manager import CacheManager
    m = CacheManager([_need(6, 3)], 4, 20, 2, 64)
    m.allocate_pools("cpu", torch.float32)
    m.poison_freed = True
    s, other = m.acquire(), m.acquire()
    m.reserve(s, 13)
    m.reserve(other, 13)
    mine, theirs = m.groups[1].tables[s][0], m.groups[1].tables[other][0]
    m.release(s)
    assert torch.isnan(m.pools[0]["k_block"][mine]).all() and torch.isnan(m.pools[0]["v_block"][mine]).all()
    assert not torch.isnan(m.pools[0]["k_block"][theirs]).any()


@pytest.mark.parametrize("window,block,page", [(5, 9, 4), (1, 1, 2), (7, 3, 1), (16, 16, 8), (3, 12, 16)])
def test_a_blocks_tokens_stay_cached_until_its_mean_is_formed(window, block, page):
    """At every length, the pages of the block under way and of the next row's window are held."""
    from ninfer_amd.cache.manager import CacheManager
    m = CacheManager([_need(max(window, block), block)], page, 200, 1, 120)
    s = m.acquire()
    for n in range(1, 100):
        m.reserve(s, n)
        m.commit(s, n)
        for p in list(range(n // block * block, n)) + list(range(max(0, n - window + 1), n)):
            assert m.groups[0].tables[s][p // page] >= 0, (n, p)
        assert len(m.groups[1].tables[s]) == -(-(n // block) // page)


# ---- the plain implementation's own properties -----------------------------------------------

def test_plain_blocks_by_hand():
    vis = plain.visible_blocks(12, 4, 3)
    assert vis.shape == (12, 4)
    # block b ends at 3 b + 2 and is seen from row 3 b + 6 on
    assert [int(v.sum()) for v in vis] == [0] * 6 + [1] * 3 + [2] * 3
    assert plain.visible_blocks(3, 1, 1)[2].tolist() == [True, True, False]
    x = torch.arange(14, dtype=D).reshape(7, 1, 2)
    assert torch.equal(plain.block_means(x, 3), torch.tensor([[[2.0, 3.0]], [[8.0, 9.0]]], dtype=D))
    # one softmax over blocks and keys: with equal scores the weights are equal
    n, window, pool = 10, 4, 3
    q = torch.zeros(n, 1, 2, dtype=D)
    v = torch.arange(n, dtype=D).reshape(n, 1, 1)
    out = plain.attend(q, torch.zeros(n, 1, 2, dtype=D), v, 1.0, window, pool)
    assert torch.allclose(out[9, 0, 0], torch.tensor((1 + 4 + 6 + 7 + 8 + 9) / 6, dtype=D))
    assert torch.allclose(out[5, 0, 0], torch.tensor((2 + 3 + 4 + 5) / 4, dtype=D))    # 0 and 1 are not seen


def test_plain_frequencies_ramp_and_pairings():
    r = {"base": 100.0, "dims": 8, "scaling": {"factor": 4.0, "original": 40, "fast": 3.0, "slow": 0.25}}
    f, mag = plain.frequencies(r)
    base = [100.0 ** (-2 * i / 8) for i in range(4)]
    at = [8 * math.log(40 / (2 * math.pi * t)) / (2 * math.log(100.0)) for t in (3.0, 0.25)]
    lo, hi = math.floor(at[0]), math.ceil(at[1])
    assert (lo, hi) == (0, 3) and abs(mag - (1 + 0.1 * math.log(4.0))) < 1e-15
    for i in range(4):
        ramp = i / 3
        assert abs(f[i] - (base[i] / 4 * ramp + base[i] * (1 - ramp))) < 1e-15
    one, m1 = plain.frequencies({"base": 100.0, "dims": 8})
    assert m1 == 1.0 and torch.allclose(one, torch.tensor(base, dtype=D))
    x = torch.randn(3, 2, 10, dtype=D, generator=torch.Generator().manual_seed(2))
    pos = torch.tensor([0, 5, 9])
    for pairing in ("half", "interleaved"):
        y = plain.rotate(x, pos, r, pairing)
        assert torch.allclose(y[0, :, :8], mag * x[0, :, :8]) and torch.equal(y[..., 8:], x[..., 8:])
        assert torch.allclose(y[..., :8].norm(dim=-1), mag * x[..., :8].norm(dim=-1))
    a = 5 * float(f[1])
    y = plain.rotate(x, pos, r, "interleaved")[1, 0]
    assert abs(y[2] - mag * (x[1, 0, 2] * math.cos(a) - x[1, 0, 3] * math.sin(a))) < 1e-12
    y = plain.rotate(x, pos, r, "half")[1, 0]
    assert abs(y[5] - mag * (x[1, 0, 5] * math.cos(a) + x[1, 0, 1] * math.sin(a))) < 1e-12


def test_framework_frequencies_equal_the_plain_ones():
    from ninfer_amd.parts import Rotary
    for base, dims, sc in ((300.0, 12, (3.0, 24, 4.0, 0.5)), (10000.0, 64, (8.0, 2048, 32.0, 1.0)),
                           (50.0, 16, (2.0, 4000, 64.0, 0.001)), (1e6, 8, (4.0, 48, 2.0, 2.0)),
                           (100.0, 8, (1.0, 40, 3.0, 0.25)), (10000.0, 20, None)):
        r = rudazen_cases.rot(dims, base, sc)
        part = Rotary(dims, base, scaling=r.get("scaling"))
        f, mag = plain.frequencies(r)
        assert torch.equal(part.inv_freq(), f.float()) and part.magnitude == mag


def test_plain_recurrence_by_hand_and_in_pieces():
    g = torch.Generator().manual_seed(3)
    n, H, d, dv = 9, 2, 3, 4
    q, v = torch.randn(n, H, d, generator=g, dtype=D), torch.randn(n, H, dv, generator=g, dtype=D)
    f = plain.forget_gates(torch.randn(n, H, d, generator=g, dtype=D), torch.tensor([0.0, 0.4, 0.9]))
    assert (f[..., 1] > 0.4).all() and (f[..., 2] > 0.9).all() and (f < 1).all()
    o, last = plain.gated_recurrence(q, f, v)
    first = ((1 - f[0]) * q[0]).sum(-1, keepdim=True) * v[0]
    assert torch.allclose(o[0], first)
    w2 = f[2] * f[1] * (1 - f[0])      # what is left of the first token's write at the third
    part = (w2 * q[2]).sum(-1, keepdim=True) * v[0] + (f[2] * (1 - f[1]) * q[2]).sum(-1, keepdim=True) * v[1] \
        + ((1 - f[2]) * q[2]).sum(-1, keepdim=True) * v[2]
    assert torch.allclose(o[2], part)
    a, mid = plain.gated_recurrence(q[:4], f[:4], v[:4])
    b, end = plain.gated_recurrence(q[4:], f[4:], v[4:], mid)
    assert torch.allclose(torch.cat([a, b]), o) and torch.allclose(end, last)


# ---- the engine's host logic on plain stand-ins ----------------------------------------------

@pytest.fixture(scope="module", params=list(rudazen_cases.CASES))
def host_case(request, tmp_path_factory):
    import ninfer_amd
    make, seed = rudazen_cases.CASES[request.param]
    raw = make()
    d = str(tmp_path_factory.mktemp(f"rudazen_host_{request.param}"))
    ninfer_amd.write_random_model(d, raw, seed, dtype="float32", std=STD)
    cfg, w = util.read_folder(d)
    reqs = {f"r{i}": util.random_tokens(n, raw["vocab"], seed + i) for i, n in enumerate([37, 1, 12, 50, 23])}
    return {"name": request.param, "dir": d, "cfg": raw, "reqs": reqs,
            "ref": {k: plain.forward(cfg, w, v)[0] for k, v in reqs.items()}}


def _host_runner(case, **more):
    from ninfer_amd import EngineOptions, load_model
    from plain_ops import PlainOps
    opt = dict(dtype="float32", device="cpu", max_context=64, num_sequences=4, page_size=4, num_pages=40,
               check_pages=True, poison_freed_pages=True)
    opt.update(more)
    return load_model(case["dir"], EngineOptions(**opt), ops=PlainOps())


def _close(case, got):
    for rid, g in got.items():
        torch.testing.assert_close(g.double(), case["ref"][rid.split("#")[0]], atol=2e-4, rtol=2e-4)


def test_host_every_way_of_cutting(host_case):
    runner = _host_runner(host_case)
    for rid, toks in host_case["reqs"].items():
        scheds = [util.schedule_whole(rid, toks), util.schedule_portions(rid, toks, seed=len(toks))]
        if len(toks) > 1:
            scheds.append(util.schedule_tail(rid, toks, 9))
        for sched in scheds:
            _close(host_case, util.run_schedule(runner, sched))
    assert all(g.allocator.in_use == 0 for g in runner.cache.groups)


def test_host_layer_by_layer(host_case):
    from ninfer_amd.engine import Chunk
    cfg, w = util.read_folder(host_case["dir"])
    toks = host_case["reqs"]["r4"]
    streams = plain.forward(cfg, w, toks)[1]
    runner = _host_runner(host_case)
    got = []
    runner.tap = lambda i, residual, pending: got.append(residual.clone())
    runner.step([Chunk(runner.open(), toks, [])])
    assert len(got) == len(streams)
    for g, want in zip(got, streams):
        torch.testing.assert_close(g.double(), want, atol=1e-4, rtol=1e-4)


def test_host_mixed_batches_reuse_pages_and_slots(host_case):
    """Portions beside single tokens, a pool that forces pages (of tokens and of blocks) to be
    used again, two state slots for five requests and their repeats: a slot's recurrent state
    starts at zero for every request that takes it, and the windows give their pages back."""
    runner = _host_runner(host_case, num_sequences=2, num_pages=26)
    reqs = dict(host_case["reqs"])
    reqs.update({k + "#2": v for k, v in host_case["reqs"].items()})
    _close(host_case, util.run_schedule(runner, util.schedule_mixed(reqs, seed=2, max_live=2)))
    assert all(g.allocator.reused > 0 for g in runner.cache.groups)
    assert sum(g.window_freed for g in runner.cache.groups) > 0
    runner.cache.check()


def test_host_generation_through_the_scheduler(host_case):
    """Greedy generation by the scheduler (admission, portions under a token budget, batched
    decoding with fewer slots than requests, a pool small enough to preempt), token for token
    the plain choice."""
    from ninfer_amd import Request, Sampler, SamplingParams, Scheduler
    from plain_ops import PlainOps
    cfg, w = util.read_folder(host_case["dir"])
    prompts = [host_case["reqs"]["r2"], host_case["reqs"]["r1"], host_case["reqs"]["r4"][:7],
               host_case["reqs"]["r0"][:15]]
    want = []
    for p in prompts:
        toks = list(p)
        for _ in range(6):
            z = plain.forward(cfg, w, toks)[0]
            top = torch.topk(z[-1], 2).values
            if top[0] - top[1] < 1e-3:
                break
            toks.append(int(z[-1].argmax()))
        want.append(toks[len(p):])
    runner = _host_runner(host_case, num_sequences=2, prefill_chunk=8, num_pages=8)
    sched = Scheduler(runner, Sampler(PlainOps(), runner.device))
    reqs = [Request(f"q{i}", list(p), SamplingParams.greedy(6)) for i, p in enumerate(prompts)]
    for r in reqs:
        sched.add(r)
    sched.run()
    assert all(r.status == "finished" for r in reqs), [r.error for r in reqs]
    assert [r.output[:len(x)] for r, x in zip(reqs, want)] == want


def test_host_two_mixers_inside_other_blocks(tmp_path):
    """Mixers side by side under a block that takes plain rows (their normed half sum is formed
    by itself), as another design might use them: the pre-norm block's stream is x + mixer(norm x)."""
    from ninfer_amd.parts import Attention, ForgetGateAttention, NoPosition, PreNormBlock, RMSNorm, SideBySide, SwiGLU
    from ninfer_amd.models.spec import ModelSpec
    from ninfer_amd.parts import LMHead, TokenEmbedding
    from ninfer_amd import EngineOptions
    from ninfer_amd.engine import Chunk
    from ninfer_amd.engine.runner import ModelRunner
    from ninfer_amd.weights import RandomSource
    from plain_ops import PlainOps
    names = {"q": "q", "k": "k", "v": "v", "o": "o", "g": "g", "temp": "temp", "q_norm": "q.norm", "k_norm": "k.norm"}
    left = Attention("b.left.", 24, 2, 1, 8, NoPosition(), qkv_bias=False, window=6, qk_norm_eps=1e-5,
                     qk_norm="projection", names=names, head_temp=True, output_gate=True)
    right = ForgetGateAttention("b.right.", 24, 2, 4, 6, 1e-5)
    mixer = SideBySide(left, right, "b.left.out", "b.right.out", 24, 1e-5)
    block = PreNormBlock(RMSNorm("n1.", 24, 1e-5), mixer, RMSNorm("n2.", 24, 1e-5),
                         SwiGLU("f.", 24, 16, names=("gate", "up", "down")))
    spec = ModelSpec(TokenEmbedding("e.", 50, 24), [block], RMSNorm("nf.", 24, 1e-5), LMHead("h.", 50, 24))
    src = RandomSource(spec.tensor_specs(), 5, torch.float32, std=STD)
    w = {n: src.read(n) for n in src.specs}
    runner = ModelRunner(spec, src, EngineOptions(dtype="float32", device="cpu", max_context=32, num_sequences=2,
                                                  page_size=4, check_pages=True), ops=PlainOps())
    toks = util.random_tokens(19, 50, 1)
    x = w["e.weight"].double()[torch.tensor(toks)]
    m = {"left": {"heads": 2, "kv_heads": 1, "dim": 8, "vdim": 8, "scale": 8 ** -0.5, "mask": {"size": 6}},
         "right": {"heads": 2, "dim": 4, "vdim": 6}}
    x = x + plain.side_by_side(w, "b.", m, plain.rms_norm(x, w["n1.weight"], 1e-5), 1e-5)
    x = x + plain.feed_forward(w, "f.", plain.rms_norm(x, w["n2.weight"], 1e-5))
    want = plain.lin(w, "h.weight", plain.rms_norm(x, w["nf.weight"], 1e-5))
    slot = runner.open()
    got = torch.cat([runner.step([Chunk(slot, toks[:11], list(range(11)))]),
                     runner.step([Chunk(slot, toks[11:], list(range(8)))])])
    torch.testing.assert_close(got.double(), want, atol=2e-4, rtol=2e-4)
