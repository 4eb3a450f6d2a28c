"""Nosedra without a GPU: the configuration reader, the model the builder makes (tensor names
and shapes, caches, state), parameters that are refused, the plain implementation's own
properties (frequencies, sink, gates, both recurrences in pieces, the convolution), and the
engine's host logic on plain stand-ins for the kernels."""
import copy
import math

import pytest
import torch

import nosedra_cases
import plain_nosedra as plain
import util

D = torch.float64
STD = 0.25


def _spec(raw):
    from ninfer_amd import build_spec
    return build_spec(raw)


# ---- reader and builder ----------------------------------------------------------------------

def test_reader_reads_every_key():
    cfg, _ = _spec(nosedra_cases.config_odd())
    assert (cfg.vocab, cfg.width, cfg.eps, cfg.softcap, cfg.side_dim) == (211, 72, 1e-5, 7.0, 9)
    a = cfg.layers[0].mixer
    assert (a.heads, a.vdim, a.state, a.groups, a.taps, a.norm_groups) == (6, 10, 12, 3, 3, 4)
    m = cfg.layers[1].mixer
    assert (m.left.heads, m.left.kv_heads, m.left.dim, m.left.vdim) == (6, 2, 20, 12)
    assert (m.left.rot.dims, m.left.rot.base, m.left.rot.factor) == (10, 500.0, 3.0)
    assert m.left.scale == 1 / math.sqrt(20) and (m.left_scale, m.right_scale) == (0.7, -1.3)
    assert (m.right.heads, m.right.dim, m.right.vdim, m.right.gate_cap) == (3, 14, 9, 6.0)
    assert cfg.layers[3].mixer.left.rot.factor == 1.0 and cfg.layers[3].mixer.left.scale == 0.4
    assert [x.ff for x in cfg.layers] == [40, 56, None, 24]
    ones, _ = _spec(nosedra_cases.config_ones())
    assert ones.layers[1].mixer.left.rot.dims == 0 and ones.softcap == 0.0


@pytest.mark.parametrize("change,word", [
    (lambda c: c.pop("vocab"), "vocab"),
    (lambda c: c.pop("token_side"), "token_side"),
    (lambda c: c["token_side"].update(dim=0), "dim"),
    (lambda c: c["norm"].pop("eps"), "eps"),
    (lambda c: c.update(logit_softcap=-1.0), "logit_softcap"),
    (lambda c: c["layers"][0].update(type="attention"), "type"),
    (lambda c: c["layers"][0]["mixer"].update(groups=4), "groups"),
    (lambda c: c["layers"][0]["mixer"].update(norm_groups=7), "norm_groups"),
    (lambda c: c["layers"][0]["mixer"].update(conv=0), "conv"),
    (lambda c: c["layers"][0]["mixer"].pop("state"), "state"),
    (lambda c: c["layers"][1]["mixer"]["left"].update(heads=5), "heads"),
    (lambda c: c["layers"][1]["mixer"]["left"]["rot"].update(dims=7), "rot.dims"),
    (lambda c: c["layers"][1]["mixer"]["left"]["rot"]["scaling"].update(factor=0.0), "factor"),
    (lambda c: c["layers"][1]["mixer"]["left"].update(scale=-1.0), "scale"),
    (lambda c: c["layers"][1]["mixer"]["right"].update(gate_cap=0), "gate_cap"),
    (lambda c: c["layers"][1]["mixer"].pop("right"), "right"),
    (lambda c: c["layers"][1]["mixer"].pop("left_scale"), "left_scale"),
    (lambda c: c["layers"][1]["mlp"].update(kind="moe"), "kind"),
])
def test_reader_names_the_key_it_refuses(change, word):
    from ninfer_amd.config import ConfigError
    raw = copy.deepcopy(nosedra_cases.config_odd())
    change(raw)
    with pytest.raises(ConfigError, match=word):
        _spec(raw)


@pytest.mark.parametrize("name", list(nosedra_cases.CASES))
def test_builder_names_every_tensor(name):
    raw = nosedra_cases.CASES[name][0]()
    _, spec = _spec(raw)
    specs = {k: v.shape for k, v in spec.tensor_specs().items()}
    w, side = raw["width"], raw["token_side"]["dim"]
    want = {"embed": (raw["vocab"], w), "head": (raw["vocab"], w), "final.norm": (w,),
            "side.embed": (raw["vocab"], side * len(raw["layers"]))}
    for i, layer in enumerate(raw["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        want.update({p + "norm1": (w,), p + "side.gate": (side, w), p + "side.proj": (w, side), p + "side.norm": (w,)})
        if layer["type"] == "parallel":
            a, b, q = m["left"], m["right"], p + "mix.left."
            want.update({q + "q": (a["heads"] * a["dim"], w), q + "k": (a["kv_heads"] * a["dim"], w),
                         q + "v": (a["kv_heads"] * a["vdim"], w), q + "g": (a["heads"] * a["vdim"], w),
                         q + "o": (w, a["heads"] * a["vdim"]), q + "sink": (a["heads"],)})
            q, H, qk, v = p + "mix.right.", b["heads"], b["heads"] * b["dim"], b["heads"] * b["vdim"]
            want.update({q + "q": (qk, w), q + "k": (qk, w), q + "v": (v, w), q + "g": (v, w), q + "o": (w, v),
                         q + "norm": (v,), q + "i": (H, w), q + "i.b": (H,), q + "f": (H, w), q + "f.b": (H,)})
        else:
            inner, gn = m["heads"] * m["vdim"], m["groups"] * m["state"]
            q = p + "mix."
            want.update({q + "in": (2 * inner + 2 * gn + m["heads"], w), q + "conv": (inner + 2 * gn, m["conv"]),
                         q + "conv.b": (inner + 2 * gn,), q + "norm": (inner,), q + "o": (w, inner)})
            want.update({q + n: (m["heads"],) for n in ("dt_bias", "A_log", "D")})
        if layer["mlp"]:
            ff = layer["mlp"]["ff"]
            want.update({p + "norm2": (w,), p + "mlp.gate": (ff, w), p + "mlp.gate.b": (ff,), p + "mlp.up": (ff, w),
                         p + "mlp.up.b": (ff,), p + "mlp.down": (w, ff), p + "mlp.down.b": (w,)})
    assert specs == want
    spare = {f"l{i}.norm2" for i, layer in enumerate(raw["layers"]) if not layer["mlp"]}
    assert set(spec.unused_tensor_specs()) >= spare


def test_caches_and_state():
    """Attention keeps keys and values of all positions; the memories keep their state per
    request in whole pieces of 16 bytes, so that every layer's starts at one."""
    _, spec = _spec(nosedra_cases.config_odd())
    mixers = [b.mixer for b in spec.blocks]
    need = mixers[1].cache_need()
    assert need.window is None and [(p.name, p.outer, p.inner) for p in need.pools] == [("k", (2,), (20,)), ("v", (2,), (12,))]
    assert mixers[0].cache_need() is None and mixers[2].cache_need() is None
    up4 = lambda n: -(-n // 4) * 4
    assert mixers[0].state_floats() == up4(6 * 12 * 10) + up4(2 * (60 + 72))
    assert mixers[1].state_floats() == up4(3 * (14 * 9 + 14 + 1)) and mixers[1].state_floats() % 4 == 0
    ones = [b.mixer for b in _spec(nosedra_cases.config_ones())[1].blocks]
    assert ones[0].state_floats() == 16 * 8       # one tap keeps no inputs


def test_what_the_engine_holds_reads_back_by_name():
    """Gains stored around zero, the rates, taps and stacked products read back as the checkpoint
    has them."""
    from ninfer_amd import EngineOptions
    from ninfer_amd.engine.runner import ModelRunner
    from ninfer_amd.weights import RandomSource
    from plain_ops import PlainOps
    _, spec = _spec(nosedra_cases.config_odd())
    src = RandomSource(spec.tensor_specs(), 3, torch.float32, std=STD)
    runner = ModelRunner(spec, src, EngineOptions(dtype="float32", device="cpu", max_context=16, num_sequences=1,
                                                  page_size=4), ops=PlainOps())
    assert runner.tensor_names() == sorted(src.specs)
    for n in src.specs:
        assert torch.equal(runner.tensor(n).float(), src.read(n)), n


def test_parameters_that_do_not_go_together_are_refused():
    from ninfer_amd.parts import Attention, MatrixMemory, NoPosition, Rotary, SideBySide, StateSpace, TokenSide, TokenSideTable
    base = dict(prefix="a.", hidden=16, heads=2, kv_heads=1, head_dim=8, position=NoPosition(), qkv_bias=False)
    for more in (dict(qk_norm="unit"), dict(qk_norm="unit", qk_norm_eps=1e-5, conv_taps=2), dict(sink="big"),
                 dict(sink="learned", qkv_bias=True), dict(sink="learned", own_kv=False),
                 dict(qk_norm="unit", qk_norm_eps=1e-5, position=Rotary(8, 100.0, scaling=dict(
                     factor=2.0, original=8, fast=4.0, slow=1.0)))):
        with pytest.raises(ValueError):
            Attention(**{**base, **more})
    left, right = Attention(**base, output_gate=True), MatrixMemory("m.", 16, 2, 4, 4, 8.0, 1e-5)
    for more in (dict(left_norm="x"), dict(left_norm="x", right_norm="y", left_factor=0.5)):
        with pytest.raises(ValueError):
            SideBySide(left, right, hidden=16, **more)
    for bad in (lambda: MatrixMemory("m.", 16, 2, 4, 4, 0.0, 1e-5), lambda: StateSpace("s.", 16, 3, 4, 4, 2, 4, 1, 1e-5),
                lambda: StateSpace("s.", 16, 4, 4, 4, 2, 0, 1, 1e-5), lambda: TokenSide("t.", 16, TokenSideTable("e", 9, 2, 4), 2, 1e-5),
                lambda: Rotary(8, 100.0, scaling={"factor": 0.0})):
        with pytest.raises(ValueError):
            bad()


# ---- the plain implementation's own properties -----------------------------------------------

def test_framework_frequencies_equal_the_plain_ones():
    from ninfer_amd.parts import Rotary
    for base, dims, factor in ((300.0, 12, 3.0), (10000.0, 64, 8.0), (50.0, 16, 0.5), (1e6, 2, 1.0)):
        f = Rotary(dims, base, scaling={"factor": factor}).inv_freq()
        x = torch.zeros(1, 1, dims, dtype=D)
        x[..., :dims // 2] = 1.0
        y = plain.rotate(x, torch.tensor([1]), {"base": base, "dims": dims, "scaling": {"factor": factor}})
        assert torch.allclose(torch.atan2(y[0, 0, dims // 2:], y[0, 0, :dims // 2]), f.double(), atol=1e-7)


def test_plain_rotation_and_unit_heads():
    x = torch.randn(3, 2, 10, dtype=D, generator=torch.Generator().manual_seed(2))
    rot = {"base": 100.0, "dims": 8, "scaling": {"factor": 2.0}}
    y = plain.rotate(x, torch.tensor([0, 5, 9]), rot)
    assert torch.equal(y[0], x[0]) and torch.equal(y[..., 8:], x[..., 8:])
    a = 5 * 100.0 ** (-2 / 8) / 2
    assert abs(y[1, 0, 5] - (x[1, 0, 5] * math.cos(a) + x[1, 0, 1] * math.sin(a))) < 1e-12
    # turned first or brought to unit size first is the same
    assert torch.allclose(plain.unit(y, 1e-3), plain.rotate(plain.unit(x, 1e-3), torch.tensor([0, 5, 9]), rot))


def test_plain_sink_by_hand():
    n = 4
    q, v = torch.zeros(n, 2, 3, dtype=D), torch.arange(1.0, n + 1, dtype=D).reshape(n, 1, 1)
    out = plain.attend(q, torch.zeros(n, 1, 3, dtype=D), v, 0.5, torch.tensor([math.log(2.0), -60.0]))
    for i in range(n):   # equal scores of 0: each key counts 1, the sink e^(its score)
        total = sum(range(1, i + 2))
        assert abs(out[i, 0, 0] - total / (i + 1 + 2)) < 1e-6 and abs(out[i, 1, 0] - total / (i + 1)) < 1e-12


def test_plain_memory_by_hand_and_in_pieces():
    g = torch.Generator().manual_seed(3)
    n, H, d, dv = 9, 2, 3, 4
    q, k, v = (torch.randn(n, H, x, generator=g, dtype=D) for x in (d, d, dv))
    write = torch.randn(n, H, generator=g, dtype=D) * 3
    keep = plain.log_sigmoid(torch.randn(n, H, generator=g, dtype=D) * 2)
    o, (S, z, m) = plain.memory(q, k, v, write, keep)
    # the stabiliser cancels but for the floor: in numbers without it
    for h in range(H):
        T, u = torch.zeros(d, dv, dtype=D), torch.zeros(d, dtype=D)
        for t in range(n):
            T = keep[t, h].exp() * T + write[t, h].exp() * torch.outer(k[t, h], v[t, h])
            u = keep[t, h].exp() * u + write[t, h].exp() * k[t, h]
            want = T.T @ q[t, h] / max(abs(float(u @ q[t, h])), 1.0)
            assert torch.allclose(o[t, h], want, rtol=1e-3, atol=1e-6)
        assert torch.allclose(S[h] * m[h].exp(), T) and torch.allclose(z[h] * m[h].exp(), u)
    # m starts at 0: a first write gate below it leaves it there but for the forget gate
    low = torch.full((1, H), -9.0, dtype=D)
    assert torch.equal(plain.memory(q[:1], k[:1], v[:1], low, keep[:1])[1][2], torch.maximum(keep[0], low[0]))
    a, mid = plain.memory(q[:4], k[:4], v[:4], write[:4], keep[:4])
    b, end = plain.memory(q[4:], k[4:], v[4:], write[4:], keep[4:], mid)
    assert torch.allclose(torch.cat([a, b]), o) and all(torch.allclose(x, y) for x, y in zip(end, (S, z, m)))


def test_plain_state_space_by_hand_and_in_pieces():
    g = torch.Generator().manual_seed(4)
    n, H, dv, G, N = 7, 4, 3, 2, 5
    x, B, C = (torch.randn(n, *s, generator=g, dtype=D) for s in ((H, dv), (G, N), (G, N)))
    dt, rate = plain.softplus(torch.randn(n, H, generator=g, dtype=D)), torch.tensor([0.1, 1.0, 3.0, 0.0], dtype=D)
    y, S = plain.state_space(x, B, C, dt, rate)
    for h in range(H):
        for t in range(n):
            want = sum(torch.exp(-rate[h] * dt[j + 1:t + 1, h].sum()) * dt[j, h] * (B[j, h // 2] @ C[t, h // 2]) * x[j, h]
                       for j in range(t + 1))
            assert torch.allclose(y[t, h], want)
    a, mid = plain.state_space(x[:3], B[:3], C[:3], dt[:3], rate)
    b, end = plain.state_space(x[3:], B[3:], C[3:], dt[3:], rate, mid)
    assert torch.allclose(torch.cat([a, b]), y) and torch.allclose(end, S)


def test_plain_convolution_and_activations_by_hand():
    x = torch.arange(1.0, 6.0, dtype=D)[:, None]
    y = plain.causal_conv(x, torch.tensor([[2.0, 3.0, 5.0]]), torch.tensor([10.0]))
    assert y[:, 0].tolist() == [15.0, 23.0, 33.0, 43.0, 53.0]
    z = torch.tensor([-40.0, -1.0, 0.0, 2.0, 40.0], dtype=D)
    assert torch.allclose(plain.softplus(z), torch.nn.functional.softplus(z))
    assert torch.allclose(plain.log_sigmoid(z), torch.nn.functional.logsigmoid(z))
    assert torch.allclose(plain.gelu(z), torch.nn.functional.gelu(z, approximate="tanh"))


# ---- the engine's host logic on plain stand-ins ----------------------------------------------

@pytest.fixture(scope="module", params=list(nosedra_cases.CASES))
def host_case(request, tmp_path_factory):
    import ninfer_amd
    make, seed = nosedra_cases.CASES[request.param]
    raw = make()
    d = str(tmp_path_factory.mktemp(f"nosedra_host_{request.param}"))
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
        torch.testing.assert_close(g.double(), case["ref"][rid.split("#")[0]], atol=3e-4, rtol=3e-4)


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

    def tap(i, residual, pending):
        whole = residual.clone()
        runner.ops.stream_norm(whole, pending)
        got.append(whole)
    runner.tap = tap
    runner.step([Chunk(runner.open(), toks, [])])
    assert len(got) == len(streams)
    for g, want in zip(got, streams):
        assert (g.double() - want).abs().max() <= 5e-5 * max(1.0, want.abs().max().item())


def test_host_mixed_batches_reuse_pages_and_slots(host_case):
    """Portions beside single tokens, a pool that forces pages to be used again, two state slots
    for five requests and their repeats: recurrent states and convolution inputs start at zero
    for every request that takes a slot."""
    runner = _host_runner(host_case, num_sequences=2, num_pages=26)
    reqs = dict(host_case["reqs"])
    reqs.update({k + "#2": v for k, v in host_case["reqs"].items()})
    _close(host_case, util.run_schedule(runner, util.schedule_mixed(reqs, seed=2, max_live=2)))
    assert all(g.allocator.reused > 0 for g in runner.cache.groups)
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


@pytest.mark.parametrize("kind", ["state-space", "parallel"])
def test_host_models_of_one_kind_of_layer(kind, tmp_path):
    import ninfer_amd
    raw = nosedra_cases.alone(kind)
    ninfer_amd.write_random_model(str(tmp_path), raw, 6, dtype="float32", std=STD)
    cfg, w = util.read_folder(str(tmp_path))
    reqs = {f"r{i}": util.random_tokens(n, raw["vocab"], i) for i, n in enumerate([21, 1, 30])}
    case = {"dir": str(tmp_path), "ref": {k: plain.forward(cfg, w, v)[0] for k, v in reqs.items()}}
    runner = _host_runner(case, num_sequences=2)
    assert bool(runner.cache.groups) == (kind == "parallel")
    _close(case, util.run_schedule(runner, util.schedule_mixed(reqs, seed=5, max_live=2)))


def test_host_new_parts_inside_other_blocks():
    """A state-space layer and a pair of mixers without output norms under a block that takes
    plain rows, and a matrix memory by itself, as another design might use them: every layer is
    x + rms(mixer(rms(x) g)) g'."""
    from ninfer_amd import EngineOptions
    from ninfer_amd.engine import Chunk
    from ninfer_amd.engine.runner import ModelRunner
    from ninfer_amd.models.spec import ModelSpec
    from ninfer_amd.parts import (Attention, LMHead, MatrixMemory, NoPosition, OutputRMSNorm, RMSNorm, SandwichBlock,
                                  SideBySide, StateSpace, TokenEmbedding)
    from ninfer_amd.weights import RandomSource
    from plain_ops import PlainOps
    names = {k: k for k in ("q", "k", "v", "o", "g", "sink")}
    eps, w_ = 1e-5, 24

    def memory(p):
        return MatrixMemory(p, w_, 2, 4, 6, 8.0, eps)
    left = Attention("m1.left.", w_, 2, 1, 8, NoPosition(), qkv_bias=False, qk_norm="unit", qk_norm_eps=eps,
                     sink="learned", output_gate=True, names=names)
    mixers = [StateSpace("m0.", w_, 4, 3, 5, 2, 3, 2, eps),
              SideBySide(left, memory("m1.right."), hidden=w_, left_factor=0.7, right_factor=-1.2), memory("m2.")]
    blocks = [SandwichBlock(RMSNorm(f"a{i}.", w_, eps), m, OutputRMSNorm(f"b{i}", w_, eps, single_gain=False))
              for i, m in enumerate(mixers)]
    spec = ModelSpec(TokenEmbedding("e.", 50, w_), blocks, RMSNorm("nf.", w_, eps), LMHead("h.", 50, w_))
    src = RandomSource(spec.tensor_specs(), 5, torch.float32, std=STD)
    w = {n: src.read(n) for n in src.specs}
    runner = ModelRunner(spec, src, EngineOptions(dtype="float32", device="cpu", max_context=32, num_sequences=2,
                                                  page_size=4, check_pages=True), ops=PlainOps())
    toks = util.random_tokens(19, 50, 1)
    m = {"left": {"heads": 2, "kv_heads": 1, "dim": 8, "vdim": 8, "scale": 8 ** -0.5},
         "right": {"heads": 2, "dim": 4, "vdim": 6, "gate_cap": 8.0}, "left_scale": 0.7, "right_scale": -1.2}
    runs = [lambda h: plain.mamba2(w, "m0.", {"heads": 4, "vdim": 3, "state": 5, "groups": 2, "norm_groups": 2}, h, eps),
            lambda h: plain.side_by_side(w, "m1.", m, h, eps), lambda h: plain.matrix_memory(w, "m2.", m["right"], h, eps)]
    x = w["e.weight"].double()[torch.tensor(toks)]
    for i, run in enumerate(runs):
        h = plain.unit(x, eps) * w[f"a{i}.weight"].double()
        x = x + plain.unit(run(h), eps) * w[f"b{i}"].double()
    want = plain.lin(w, "h.weight", plain.unit(x, eps) * w["nf.weight"].double())
    slot = runner.open()
    got = torch.cat([runner.step([Chunk(slot, toks[:11], list(range(11)))]),
                     runner.step([Chunk(slot, toks[11:], list(range(8)))])])
    torch.testing.assert_close(got.double(), want, atol=2e-4, rtol=2e-4)
