"""Zudusun on the GPU: every kernel of its parts alone against the plain implementation's function of the same mechanism
(float32 and bfloat16): memories with a decay for every key channel, with one number a head and with one that is the same
for every token, over steps cut anywhere in slots that others left full, token by token and chunk by chunk, with decays
from none to at once; attention with a one in its denominator and keys made to stand out just inside and just outside
the window, far away, at page borders and at the first token; experts without gates on every path; the engine under
every way of cutting, recorded decoding, generation through the entry point and the scheduler, the replay program and
the command line."""
import json
import os
import subprocess
import sys
from types import SimpleNamespace

import numpy as np
import pytest
import torch

import plain_zudusun as P
import schedules
import zudusun_cases as zc
from test_zudusun_cpu import TOL, _expected, _greedy, step_through
from transformers_neuronx_amd.engine import StepEntry
from transformers_neuronx_amd.engine.batch import build_context

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
DTYPES = [("float32", torch.float32, 5e-6), ("bfloat16", torch.bfloat16, 1.2e-2)]
F64 = torch.float64


def _ops(dtype):
    from transformers_neuronx_amd.kernels import make_ops
    return make_ops("hip", dtype, DEV)


def _ctx(runs, cached, slots, tables=None, page_size=16, planners=None):
    entries = [StepEntry(i, [0] * n, []) for i, n in enumerate(runs)]
    tables = tables if tables is not None else {}
    return build_context(entries, cached, slots, {k: np.asarray(v, dtype=np.int32) for k, v in tables.items()},
                         page_size, DEV, planners)


def _close(got, want, tol, scale=None):
    """`scale`: what the difference is measured by, where `want` is a few numbers of many (the largest of all)."""
    want = want.to(F64)
    scale = float(want.abs().max()) if scale is None else float(scale)
    err = float((got.double().cpu() - want).abs().max() / max(1e-30, scale))
    assert err < tol, err


# steps of a request in slot 2 and, from the third step on, of another in slot 0. Runs of one token, of a few, just under
# and at the length from which they go by chunks here, at and around whole chunks and blocks of 16 tokens, and long ones.
CUTS0 = (0, 1, 2, 4, 5, 6, 29, 53, 54, 118, 181, 246, 247, 439, 440, 611)
CUTS1 = (None, None, 0, 1, 2, 9, 11, 12, 76, 78, 141, 142, 143, None, None, None)


def _steps():
    for s in range(len(CUTS0) - 1):
        step = [(0, CUTS0[s], CUTS0[s + 1], 2)]
        if CUTS1[s] is not None and CUTS1[s + 1] is not None:
            step.append((1, CUTS1[s], CUTS1[s + 1], 0))
        yield step


def _plan(run_lens, cached, page_size):
    from transformers_neuronx_amd.kernels.memory_plan import memory_plan
    return memory_plan(run_lens, cached, page_size, least=24)


BY_CHUNKS = {"memory": _plan}
LENGTHS = {0: CUTS0[-1], 1: 143}


# ---------------------------------------------------------------- the memories

@pytest.mark.parametrize("sizes", [
    # heads, n, v, the level of the decays' pre-activations, tau: gentle (as trained models), mixed, at once
    (1, 1, 1, 0.0, 1.0), (4, 16, 24, 2.0, 16.0), (3, 10, 7, 0.0, 1.0), (2, 64, 64, -3.0, 0.5), (6, 128, 40, 3.0, 16.0),
    (2, 256, 20, 1.0, 4.0), (2, 100, 16, -40.0, 1.0), (1, 200, 5, -6.0, 0.5), (5, 33, 5, 4.0, 8.0), (4, 48, 64, 0.0, 2.0)])
@pytest.mark.parametrize("by_chunks", [True, False])
def test_memories_with_a_decay_for_every_key_channel(sizes, by_chunks):
    """The recurrence over steps of 1, 2 and more tokens, two requests side by side in slots that former holders left
    full, every step of single tokens run twice (a recorded step is), against the whole sequence token by token."""
    heads, n, v, level, tau = sizes
    ops = _ops(torch.float32)
    ops.memory_by_chunks = by_chunks
    g = torch.Generator().manual_seed(4)
    qk, inner, before = heads * n, heads * v, 4
    rows, decay, want = {}, {}, {}
    for r, t in LENGTHS.items():
        rows[r] = torch.randn(t, before + 2 * qk + inner + 3, generator=g)
        decay[r] = (P.log_sigmoid(torch.randn(t, qk, generator=g, dtype=F64) * 2 + level) / tau).float()
        d = rows[r].double()
        q, k = d[:, before:before + qk].view(t, heads, n), d[:, before + qk:before + 2 * qk].view(t, heads, n)
        val = d[:, before + 2 * qk:before + 2 * qk + inner].view(t, heads, v)
        want[r] = P.decaying_memory(q, k, val, decay[r].double().view(t, heads, n)).reshape(t, inner)
    memory = torch.full((3, 2, heads, v, n), 3.0, device=DEV)
    for step in _steps():
        u = torch.cat([rows[r][a:b] for r, a, b, _ in step]).to(DEV)
        ld = torch.cat([decay[r][a:b] for r, a, b, _ in step]).to(DEV)
        ctx = _ctx([b - a for _, a, b, _ in step], [a for _, a, _, _ in step], [slot for _, _, _, slot in step],
                   planners=BY_CHUNKS)
        for _ in range(2 if all(b - a == 1 for _, a, b, _ in step) else 1):
            got = ops.linear_memory(u[:, before:before + 2 * qk + inner], 0, qk, 2 * qk, heads, heads, n, v, ld, None, ctx,
                                    memory, False)
        at = 0
        for r, a, b, _ in step:
            _close(got[at:at + b - a], want[r][a:b], 1e-5, want[r].abs().max())
            at += b - a
    assert float(memory[1].min()) == 3.0 and float(memory[1].max()) == 3.0       # a slot of no one is not touched


@pytest.mark.parametrize("sizes", [(1, 1, 1), (3, 10, 7), (2, 64, 64), (4, 128, 40), (2, 256, 20), (5, 33, 48)])
@pytest.mark.parametrize("by_chunks", [True, False])
def test_memories_with_a_decay_that_is_the_same_for_every_token(sizes, by_chunks):
    heads, n, v = sizes
    ops = _ops(torch.float32)
    ops.memory_by_chunks = by_chunks
    g = torch.Generator().manual_seed(5)
    qk, inner = heads * n, heads * v
    decay = torch.log(torch.tensor([0.97, 1.0, 0.9995, 0.5, 1e-9][:heads]))
    rows, want = {}, {}
    for r, t in LENGTHS.items():
        rows[r] = torch.randn(t, 2 * qk + inner, generator=g)
        d = rows[r].double()
        want[r] = P.decaying_memory(d[:, :qk].view(t, heads, n), d[:, qk:2 * qk].view(t, heads, n), d[:, 2 * qk:].view(t, heads, v),
                                    decay.double()[None, :, None].expand(t, heads, n)).reshape(t, inner)
    memory = torch.full((3, 2, heads, v, n), -2.0, device=DEV)
    for step in _steps():
        u = torch.cat([rows[r][a:b] for r, a, b, _ in step]).to(DEV)
        ctx = _ctx([b - a for _, a, b, _ in step], [a for _, a, _, _ in step], [slot for _, _, _, slot in step],
                   planners=BY_CHUNKS)
        for _ in range(2 if all(b - a == 1 for _, a, b, _ in step) else 1):
            got = ops.linear_memory(u, 0, qk, 2 * qk, heads, heads, n, v, decay.to(DEV), None, ctx, memory, False)
        at = 0
        for r, a, b, _ in step:
            _close(got[at:at + b - a], want[r][a:b], 1e-5, want[r].abs().max())
            at += b - a


def test_a_channel_that_remembers_beside_one_that_forgets():
    """Channel 0 hardly forgets: the last token reads along it what one token far back wrote, the keys between having
    nothing there. Channel 1 forgets at once: reading along it gives the present token's write alone. Channel 2 forgets
    at one token only, inside a block of 16, between a block's end and the next, or in the chunk before."""
    n, v, t = 48, 16, 400
    for at in (133, 143, 144, 200, 390):
        g = torch.Generator().manual_seed(at)
        k = torch.randn(t, n, generator=g)
        k[:, :3] = 0
        k[3, 0], k[5, 2] = 1.0, 1.0
        k[:, 1] = 1.0
        q = torch.randn(t, n, generator=g) * 0.1
        q[-1] = 0
        val = torch.randn(t, v, generator=g)
        ld = -torch.rand(t, n, generator=g) * 0.05
        ld[:, 0], ld[:, 1], ld[:, 2] = -1e-6, -60.0, 0.0
        ld[at, 2] = -2.0
        u = torch.cat([q, k, val], dim=1)
        for channel, want in ((0, val[3] * np.exp(-1e-6 * (t - 4))), (1, val[-1]), (2, val[5] * np.exp(-2.0))):
            u[-1, :3] = 0
            u[-1, channel] = 1.0
            d = u.double()
            plain = P.decaying_memory(d[:, None, :n], d[:, None, n:2 * n], d[:, None, 2 * n:], ld.double()[:, None]).view(t, v)
            assert torch.allclose(plain[-1], want.double(), atol=1e-6)
            for chunks, cuts in ((True, (0, t)), (False, (0, t)), (True, (0, 130, t - 1, t))):
                ops = _ops(torch.float32)
                ops.memory_by_chunks = chunks
                memory = torch.full((1, 2, 1, v, n), 9.0, device=DEV)
                got = torch.cat([ops.linear_memory(u[a:b].to(DEV), 0, n, 2 * n, 1, 1, n, v, ld[a:b].to(DEV), None,
                                                   _ctx([b - a], [a], [0], planners=BY_CHUNKS), memory, False)
                                 for a, b in zip(cuts[:-1], cuts[1:])])
                _close(got, plain, 1e-5)
                _close(got[-1], plain[-1], 4e-5)       # (a float32 state that loses 1e-6 of itself 400 times)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("sizes", [(1, 1, 1), (1, 4096, 16), (7, 300, 5), (8, 2048, 20), (100, 513, 33), (2000, 1000, 16), (3, 70000, 2)])
def test_decays_through_the_bottleneck(sizes, dtype):
    t, channels, rank = sizes
    ops = _ops(dtype)
    g = torch.Generator().manual_seed(rank)
    rows = torch.randn(t, rank + 9, generator=g) * 3
    w, bias = (torch.randn(channels, rank, generator=g)).to(dtype), torch.randn(channels, generator=g) * 4
    want = P.log_sigmoid(rows[:, 5:5 + rank].double() @ w.double().T + bias.double()) / 7.0
    got = ops.channel_decays(rows.to(DEV)[:, 5:5 + rank], w.to(DEV), bias.to(DEV), 7.0)
    _close(got, want, 1e-6)
    near_zero = (want.abs() < 1e-3) & (want.abs() > 1e-12)       # a decay of almost one keeps its digits
    if bool(near_zero.any()):
        assert float(((got.double().cpu() - want).abs() / want.abs())[near_zero].max()) < 1e-4


def test_the_logarithm_of_a_decay_keeps_its_digits():
    """From pre-activations of -80 (the decay is almost 0) to 80 (almost 1: the logarithm is tiny)."""
    z = torch.linspace(-80, 80, 40001)
    want = P.log_sigmoid(z.double())
    got = _ops(torch.float32).channel_decays(torch.zeros(1, 1, device=DEV), torch.zeros(z.numel(), 1, device=DEV), z.to(DEV), 1.0)
    assert float(((got[0].double().cpu() - want) / want).abs().max()) < 1e-6


@pytest.mark.parametrize("interleaved", [True, False])
@pytest.mark.parametrize("sizes", [(1, 1, 2, 2), (5, 6, 24, 10), (33, 4, 64, 64), (9, 3, 250, 200), (2, 2, 256, 256)])
def test_heads_turned_in_place(sizes, interleaved):
    t, heads, n, dims = sizes
    ops = _ops(torch.float32)
    x = torch.randn(t, heads * n + 11, generator=torch.Generator().manual_seed(1))
    freqs = P.frequencies(10000.0, dims).float()
    cached = 2000
    turn = P.turn_neighbours if interleaved else P.turn_halves
    want = x.double().clone()
    want[:, 3:3 + heads * n] = turn(x[:, 3:3 + heads * n].double().view(t, heads, n), torch.arange(cached, cached + t), 10000.0,
                                    dims).reshape(t, heads * n)
    dev = x.to(DEV)
    got = ops.turn_heads(dev, 3, heads, n, freqs.to(DEV), interleaved, _ctx([t], [cached], [0]))
    assert got is dev
    _close(got, want, 2e-4)                  # (float32 angles of thousands of radians)
    assert torch.equal(got.cpu()[:, :3], x[:, :3]) and torch.equal(got.cpu()[:, 3 + heads * n:], x[:, 3 + heads * n:])
    early = x.to(DEV)
    ops.turn_heads(early, 3, heads, n, freqs.to(DEV), interleaved, _ctx([t], [0], [0]))
    want[:, 3:3 + heads * n] = turn(x[:, 3:3 + heads * n].double().view(t, heads, n), torch.arange(t), 10000.0, dims).reshape(t, heads * n)
    _close(early, want, 5e-6)


@pytest.mark.parametrize("name,dtype,tol", DTYPES)
@pytest.mark.parametrize("sizes", [(1, 1, 1, 0), (7, 4, 24, 3), (33, 6, 16, 8), (9, 32, 128, 64), (3, 5, 200, 2), (6, 4, 300, 4)])
@pytest.mark.parametrize("weighted", [True, False])
def test_gate_and_norm_into_a_slice_times_a_factor(name, dtype, tol, sizes, weighted):
    t, heads, v, left = sizes
    ops = _ops(dtype)
    g = torch.Generator().manual_seed(8)
    o, rows = torch.randn(t, heads * v, generator=g) * 2, torch.randn(t, heads * v + 7, generator=g) * 2
    weight = torch.randn(heads * v, generator=g) if weighted else None
    gate = rows[:, 5:5 + heads * v]
    y = P.unit_rms(o.double().view(t, heads, v), 0.3).reshape(t, heads * v) * (1 if weight is None else weight.double())
    want = y * P.silu(gate.double())
    dev = rows.to(DEV)[:, 5:5 + heads * v]
    wd = None if weight is None else weight.to(DEV)
    _close(ops.gated_norm(o.to(DEV), dev, wd, 0.3, heads, False), want, tol)
    both = torch.full((t, left + heads * v + 4), 7.0, dtype=dtype, device=DEV)
    ops.gated_norm(o.to(DEV), dev, wd, 0.3, heads, False, out=both[:, left:left + heads * v], out_scale=-0.4)
    _close(both[:, left:left + heads * v], -0.4 * want, tol)
    assert float((both[:, :left].float() - 7).abs().sum() + (both[:, left + heads * v:].float() - 7).abs().sum()) == 0


# ---------------------------------------------------------------- attention with a window and a one in the denominator

@pytest.mark.parametrize("name,dtype,tol", [("float32", torch.float32, 4e-5), ("bfloat16", torch.bfloat16, 4e-2)])
@pytest.mark.parametrize("case", [
    # query heads, kv heads, key size, value size, cached size, length, the step's tokens, page, window, the standing-out
    # key's distance from the last query
    dict(h=4, g=2, n=16, v=16, d=16, length=300, run=1, ps=16, window=300, back=299),    # the very first token, just inside
    dict(h=4, g=2, n=16, v=16, d=16, length=300, run=1, ps=16, window=299, back=299),    # just outside
    dict(h=2, g=1, n=64, v=32, d=64, length=700, run=1, ps=64, window=137, back=136),    # decoded: the last the window keeps
    dict(h=2, g=1, n=64, v=32, d=64, length=700, run=1, ps=64, window=137, back=137),    # and the next one
    dict(h=2, g=1, n=64, v=32, d=64, length=700, run=300, ps=64, window=137, back=136),  # the same in a prompt
    dict(h=2, g=1, n=64, v=32, d=64, length=700, run=300, ps=64, window=137, back=137),
    dict(h=6, g=1, n=96, v=80, d=96, length=400, run=37, ps=64, window=81, back=80),     # at a page's border
    dict(h=6, g=1, n=96, v=80, d=96, length=400, run=37, ps=64, window=80, back=80),
    dict(h=6, g=3, n=16, v=24, d=32, length=64, run=64, ps=16, window=64, back=63),      # a whole prompt
    dict(h=1, g=1, n=64, v=64, d=64, length=129, run=2, ps=64, window=1, back=1),        # a window of one token
    dict(h=1, g=1, n=64, v=64, d=64, length=129, run=2, ps=64, window=2, back=1),
    dict(h=8, g=2, n=128, v=128, d=128, length=280, run=200, ps=64, window=None, back=279),   # no window: far away
    dict(h=4, g=2, n=64, v=128, d=128, length=530, run=1, ps=64, window=None, back=529),      # no window, decoded
    dict(h=4, g=2, n=160, v=144, d=160, length=300, run=140, ps=16, window=201, back=200),
    dict(h=4, g=2, n=32, v=32, d=32, length=330, run=130, ps=48, window=65, back=64),    # pages that are no power of two
])
@pytest.mark.parametrize("kernel", ["matrix unit", "shared out", "one set", "general"])
def test_attention_finds_the_key_that_stands_out_inside_its_window(name, dtype, tol, case, kernel):
    if kernel != "general" and dtype == torch.float32:
        pytest.skip("float32 has the one kernel")
    from transformers_neuronx_amd.kernels.attention_plan import attention_plan
    ops = _ops(dtype)
    ops.force_plain_attention = kernel == "general"
    ops.scored_decode_splits = 3 if kernel == "shared out" else 1
    ops.prefill_direct = {"one set": 2, "shared out": 3}.get(kernel, False)
    h, g, n, v, d, length, run, ps, window = (case[k] for k in ("h", "g", "n", "v", "d", "length", "run", "ps", "window"))
    standout = length - 1 - case["back"]
    gen = torch.Generator().manual_seed(7)
    proj = torch.randn(length, h * n + g * (n + v), generator=gen) * 0.3
    mark = torch.randn(n, generator=gen)
    mark = mark / mark.norm() * 6.0
    proj[standout, h * n:h * n + g * n] = mark.repeat(g)
    proj[standout, h * n + g * n:] = 4.0
    proj[length - 1, :h * n] = mark.repeat(h)
    proj = proj.to(dtype).float()
    scale = 0.6
    d64 = proj.double()
    q, k = d64[:, :h * n].view(length, h, n), d64[:, h * n:h * n + g * n].view(length, g, n)
    val = d64[:, h * n + g * n:].view(length, g, v)
    want = P.attend(q, k, val, scale, window, one_more=True)
    seen = case["back"] < (window or 1 << 30)
    assert (float(want[-1].min()) > 3.5) == seen               # the key that stands out decides, or is not there
    blocks = -(-length // ps)
    order = torch.randperm(blocks + 3, generator=torch.Generator().manual_seed(1))[:blocks].tolist()
    k_pages = torch.full((blocks + 3, g, ps, d), 50.0, dtype=dtype, device=DEV)
    v_pages = torch.full((blocks + 3, g, d, ps), 50.0, dtype=dtype, device=DEV)
    sink = torch.zeros(h, device=DEV)
    for a, b in ((0, length - run), (length - run, length)):
        if b == a:
            continue
        ctx = _ctx([b - a], [a], [0], {"g": [order]}, ps, {"attention": attention_plan})
        qd = ops.qkv_prepare(proj[a:b].to(DEV), h, g, n, v, d, None, None, 0.0, None, False, scale, None, None, ctx,
                             ctx.groups["g"], k_pages, v_pages)
        both = torch.full((b - a, h * d + 8), 7.0, dtype=dtype, device=DEV)
        got = ops.attention_scored(qd, h, g, d, ctx, ctx.groups["g"], k_pages, v_pages, window=window, value_size=v, sink=sink,
                                   out=both[:, 8:], out_scale=0.5)
        _close(got.reshape(b - a, h, d)[:, :, :v], 0.5 * want[a:b], tol)
        _close(got[-1].view(h, d)[:, :v], 0.5 * want[b - 1], tol)
        assert float((both[:, :8].float() - 7).abs().max()) == 0


@pytest.mark.parametrize("name,dtype,tol", [("float32", torch.float32, 2e-5), ("bfloat16", torch.bfloat16, 2.5e-2)])
@pytest.mark.parametrize("kind", ["attention", "left"])
def test_attention_mixers_alone(name, dtype, tol, kind):
    """The mixers as the model builds them (norms before the turn, biases, the one in the denominator, unequal heads;
    the one without any of these, whose sizes would not call for the float32 route), prompts, portions, single tokens."""
    from transformers_neuronx_amd.engine.batch import context_from
    m = dict(zc.attention(4, 2, 32, 48, 0.3, 21, 100.0, 20)[1]) if kind == "attention" else None
    layers = [zc.layer(zc.attention(4, 2, 32, 48, 0.3, 21, 100.0, 20), None)] if kind == "attention" else \
        [zc.layer(zc.parallel((4, 2, 32, 32, 0.3), (1, 16, 16, 4.0, 4), (0.8, 0.0)), None)]
    cfg = zc.ZudusunConfig.from_dict(dict(architecture="Zudusun", vocab=50, width=64, norm=dict(eps=1e-4), layers=layers, init_std=0.3))
    w = zc.weights(cfg, 3, dtype)
    if kind == "attention":
        for b in ("q.b", "k.b", "v.b", "o.b"):
            w["l0.mix." + b] = w["l0.mix." + b] * 3
    runner = zc.runner(cfg, w, dtype="float32" if dtype == torch.float32 else "bfloat16", kernels="hip", device=DEV)
    mixer = runner.model.layers[0].mixer
    h = torch.randn(90, 64, generator=torch.Generator().manual_seed(2)).to(dtype)
    wide = P.widen(w)
    want = (P.attention(m, wide, "l0.mix.", h.double(), 1e-4) if kind == "attention"
            else 0.8 * P.softmax_side(cfg.layers[0]["mixer"]["left"], wide, "l0.mix.left.", h.double()))
    if kind == "left":
        # (the other mixer's part is there with the factor 0)
        assert mixer.right_scale == 0.0
    got, at = [], 0
    for n in (1, 2, 40, 1, 1, 30, 15):
        packed = runner.prepare([StepEntry("r", [0] * n, [])])
        ctx = context_from(packed, torch.from_numpy(packed.flat).to(DEV))
        got.append(mixer.forward(h[at:at + n].to(DEV), ctx, runner.cache.caches[0], None))
        runner.cache.advance("r", n)
        at += n
    _close(torch.cat(got), want, tol)


# ---------------------------------------------------------------- the mixture

@pytest.mark.parametrize("name,dtype,tol", DTYPES)
@pytest.mark.parametrize("sizes", [
    # tokens, experts, a token's experts, width, inner size, the shared expert's inner size
    (1, 3, 1, 64, 16, 24), (37, 5, 3, 96, 40, 8), (130, 7, 7, 192, 72, 96), (9, 6, 4, 50, 30, 21), (300, 60, 6, 128, 24, 0),
    (900, 6, 4, 128, 64, 64), (700, 1, 1, 64, 32, 32), (40, 100, 5, 32, 8, 16), (8, 16, 2, 1024, 512, 256), (600, 3, 1, 64, 40, 0)])
@pytest.mark.parametrize("forced", [None, "ours", "plain"])
def test_experts_without_gates_beside_a_shared_one_with_a_number(name, dtype, tol, sizes, forced):
    """`forced`: None, as the engine would (steps of many pairs an expert through the vendor library); "ours": the one
    launch of ours at any size; "plain": without the matrix unit."""
    from transformers_neuronx_amd.parts.feed_forward import ExpertMixture
    tokens, experts, top, width, inner, shared = sizes
    if forced and (dtype == torch.float32 or (forced == "ours" and tokens < 100)):
        pytest.skip("the same path as unforced")
    ops = _ops(dtype)
    ops.expert_library_rows = 96 if forced is None else 0
    ops.expert_plain_products = forced == "plain"
    g = torch.Generator().manual_seed(5)
    part = ExpertMixture(width, experts, top, inner, "router", "e{}.", ("up", "down"), score="softmax", renormalize=True,
                         weight_on="output", activation="relu2", gated=False, router_bias_name="router.b", shared_inner=shared,
                         shared_gate_name="sg")
    w = {d.name: (torch.randn(d.shape, generator=g) * (2.0 / d.shape[-1] ** 0.5)).to(dtype) for d in part.param_decls("p.")}
    w["p.router.b"] = torch.randn(experts, generator=g)
    part.load({k: v.to(DEV) for k, v in w.items()}, "p.", ops, dtype)
    h = torch.randn(tokens, width, generator=g).to(dtype)
    residual = torch.randn(tokens, width, generator=g)
    wide = P.widen(w)
    z = h.double() @ wide["p.router"].T + wide["p.router.b"]
    chosen, weight = P.route(z, top)
    # only tokens whose choice float64 and float32 cannot see differently
    ranked = torch.sort(z, dim=-1, descending=True).values
    clear = torch.ones(tokens, dtype=torch.bool) if top == experts else (ranked[:, top - 1] - ranked[:, top]) > 1e-4
    assert int(clear.sum()) >= max(1, tokens // 2)
    assert tokens < 30 or top == experts or P.route(z - wide["p.router.b"], top)[0].tolist() != chosen.tolist()   # the bias matters
    at = part.router_at
    got_chosen, got_weight = ops.route(ops.linear(h.to(DEV), part.w_in, part.b_in, out_f32=True)[:, at:at + experts], top,
                                       "softmax", True)
    if top < experts:
        assert sorted(map(sorted, got_chosen.cpu()[clear].tolist())) == sorted(map(sorted, chosen[clear].tolist()))
    assert torch.allclose(got_weight.sum(-1).cpu(), torch.ones(tokens), atol=1e-5)
    mlp = dict(router=dict(experts=experts, top=top), expert=dict(ff=inner), shared=dict(ff=shared) if shared else None)
    want = P.mixture(mlp, wide, "p.", h.double())
    got = part.forward(h.to(DEV), SimpleNamespace(length_bound=None), residual.to(DEV))
    _close(got.cpu()[clear], (residual.double() + want)[clear], tol)
    if not shared:
        alone = part.forward(h.to(DEV), SimpleNamespace(length_bound=None), None)
        _close(alone.cpu()[clear], want[clear], tol)


@pytest.mark.parametrize("name,dtype,tol", DTYPES)
@pytest.mark.parametrize("t,f", [(1, 1), (5, 30), (9, 64), (300, 130)])
def test_an_activation_with_a_gate_number_a_row(name, dtype, tol, t, f):
    ops = _ops(dtype)
    g = torch.Generator().manual_seed(t)
    x, rows = torch.randn(t, f, generator=g) * 2, torch.randn(t, 6, generator=g) * 3
    want = P.squared_relu(x.double())
    _close(ops.row_activation(x.to(DEV), "relu2"), want, tol)
    _close(ops.row_activation(x.to(DEV), "relu2", rows.to(DEV)[:, 4:5]), want * P.sigmoid(rows[:, 4:5].double()), tol)
    for at, more in ((4, 8), (3, 5)):          # rows that lie apart, at places of a multiple of four elements and not
        wide = torch.full((t, at + f + more), 9.0)
        wide[:, at:at + f] = x
        _close(ops.row_activation(wide.to(DEV)[:, at:at + f], "relu2"), want, tol)


# ---------------------------------------------------------------- the engine

@pytest.mark.parametrize("dtype,tol", [("float32", TOL), ("bfloat16", 6e-2)])
@pytest.mark.parametrize("name", sorted(zc.CASES))
def test_schedules_on_the_gpu(name, dtype, tol):
    cfg = zc.config(name)
    w = zc.weights(cfg, 3, torch.bfloat16 if dtype == "bfloat16" else torch.float32)
    runner = zc.runner(cfg, w, dtype=dtype, kernels="hip", device=DEV, max_tokens=208)
    requests = zc.requests(cfg, [70, 33, 5, 100, 1], 1)
    expected = _expected(cfg, w, requests)
    few = 0.12 if dtype == "bfloat16" else 0.0
    for made in (schedules.whole(requests), schedules.head_then_singles(requests, tail=12), schedules.portions(requests),
                 schedules.portions(requests, sizes=(2, 2, 3, 2, 16, 2, 15, 17, 2)),
                 schedules.mixed(requests, max_tokens=208, page=16, seed=5, tail=8, max_live=3),
                 schedules.only_last(schedules.mixed(requests, max_tokens=208, page=16, seed=6, tail=20, max_live=4))):
        step_through(runner, expected, made, tol, few)
    from transformers_neuronx_amd.kernels import hip
    assert {"linear_memory", "prepare", "experts", "gemm", "scored"} <= set(hip.loaded_libraries())


@pytest.mark.parametrize("dtype,tol", [("float32", TOL), ("bfloat16", 6e-2)])
def test_long_requests_under_every_way_of_cutting(dtype, tol):
    """Requests of several chunks, windows and pages of 64."""
    cfg = zc.config("c")
    w = zc.weights(cfg, 5, torch.bfloat16 if dtype == "bfloat16" else torch.float32)
    runner = zc.runner(cfg, w, dtype=dtype, kernels="hip", device=DEV, max_tokens=1024, page_size=64)
    requests = zc.requests(cfg, [400, 129, 64, 250], 8)
    expected = _expected(cfg, w, requests)
    few = 0.12 if dtype == "bfloat16" else 0.0
    for made in (schedules.whole(requests), schedules.head_then_singles(requests, tail=20),
                 schedules.portions(requests, sizes=(100, 2, 63, 64, 81, 80, 79, 1, 128)),
                 schedules.mixed(requests, max_tokens=1024, page=64, seed=2, tail=10, max_live=4)):
        step_through(runner, expected, made, tol, few)


@pytest.mark.parametrize("name", ["a", "b", "c"])
def test_the_stream_after_every_layer_on_the_gpu(name):
    from transformers_neuronx_amd import debug
    cfg = zc.config(name)
    w = zc.weights(cfg, 2)
    toks = zc.requests(cfg, [70], 0)["r0"]
    _, layers = P.forward(cfg.to_dict(), P.widen(w), toks, return_layers=True)
    runner = zc.runner(cfg, w, dtype="float32", kernels="hip", device=DEV)
    with debug.debug_context() as taps:
        runner.step([StepEntry("r0", toks, [])])
    for i, want in enumerate(layers):
        got = taps[f"call{i}.layer{runner.model.schedule[i][0]}"]
        assert float((got.double().cpu() - want).abs().max() / want.abs().max()) < 1e-5, i


def _decode_along(runner, requests, start, joins):
    """The first `start` tokens of r0 in one step, then its tokens one by one; `joins` = {request: (from, to)}: the others
    run beside it, a token a step, from one of its positions to another."""
    got = {"r0": [runner.step([StepEntry("r0", requests["r0"][:start], list(range(start)))]).clone()],
           **{rid: [] for rid in joins}}
    for i in range(start, len(requests["r0"])):
        entries = [StepEntry("r0", [requests["r0"][i]], [0])]
        entries += [StepEntry(rid, [requests[rid][i - a]], [0]) for rid, (a, b) in joins.items() if a <= i < b]
        out = runner.step(entries)
        for row, e in enumerate(entries):
            got[e.req].append(out[row:row + 1].clone())
        for rid, (a, b) in joins.items():
            if i == b - 1:
                runner.finish(rid)
    return {rid: torch.cat(rows) for rid, rows in got.items()}


@pytest.mark.parametrize("graphs", [True, False])
def test_long_decoding_recorded_and_not(graphs):
    """300 tokens one by one beside requests that join and leave: the batch size changes (a recorded step is made for
    each), pages and slots change hands."""
    cfg = zc.config("c")
    w = zc.weights(cfg, 8)
    runner = zc.runner(cfg, w, dtype="float32", kernels="hip", device=DEV, max_tokens=512, page_size=16, use_graphs=graphs)
    requests = zc.requests(cfg, [320, 90, 60], 9)
    expected = _expected(cfg, w, requests)
    got = _decode_along(runner, requests, 20, {"r1": (50, 140), "r2": (200, 260)})
    assert (runner.graph_replays > 0) == graphs
    for rid in requests:
        assert float((got[rid].double().cpu() - expected[rid]).abs().max() / expected[rid].abs().max()) < TOL, rid


def test_long_decoding_in_bfloat16_recorded():
    cfg = zc.config("c")
    w = zc.weights(cfg, 9, torch.bfloat16)
    runner = zc.runner(cfg, w, dtype="bfloat16", kernels="hip", device=DEV, max_tokens=1024, page_size=64)
    requests = zc.requests(cfg, [600, 200], 4)
    expected = _expected(cfg, w, requests)
    got = _decode_along(runner, requests, 300, {"r1": (310, 510)})
    assert runner.graph_replays > 0
    for rid in requests:
        err = (got[rid].double().cpu() - expected[rid]).abs().amax(-1) / expected[rid].abs().max()
        assert float((err > 6e-2).double().mean()) <= 0.12, rid


@pytest.mark.parametrize("amp,tol", [("f32", TOL), ("bf16", 6e-2)])
def test_generation_through_the_entry_point(tmp_path, amp, tol):
    from safetensors.torch import load_file
    from transformers_neuronx_amd import NeuronAutoModelForCausalLM
    from transformers_neuronx_amd.weights import write_random_model
    cfg = zc.config("a")
    folder = write_random_model(cfg, str(tmp_path / "m"), 11, dtype="float32" if amp == "f32" else "bfloat16")
    w = load_file(os.path.join(folder, "model.safetensors"))
    model = NeuronAutoModelForCausalLM.from_pretrained(folder, batch_size=2, amp=amp, n_positions=64, page_size=16,
                                                       device=DEV).load()
    ids = torch.tensor([[5, 200, 17, 3], [9, 9, 100, 42]])
    logits = model(ids)
    raw, wide = cfg.to_dict(), P.widen(w)
    for row in range(2):
        want = P.forward(raw, wide, ids[row].tolist())[-1]
        assert float((logits[row].double().cpu() - want).abs().max() / want.abs().max()) < tol
    if amp == "f32":
        out = model.sample(ids, sequence_length=14, top_k=1)
        for row in range(2):
            assert out[row, 4:].tolist() == _greedy(cfg, w, ids[row].tolist(), 10)


def test_generation_through_the_scheduler_with_few_pages():
    from transformers_neuronx_amd.config import EngineConfig
    from transformers_neuronx_amd.engine.engine import LLMEngine
    from transformers_neuronx_amd.engine.factory import build_runner
    from transformers_neuronx_amd.sampling import SamplingParams
    from transformers_neuronx_amd.weights.loader import TensorDict
    cfg = zc.config("b")
    w = zc.weights(cfg, 6)
    ecfg = EngineConfig(dtype="float32", kernels="hip", device=DEV, page_size=16, max_tokens=96, max_num_seqs=3,
                        max_num_batched_tokens=24, chunk_size=9)
    engine = LLMEngine(build_runner(cfg, TensorDict(w), ecfg), ecfg)
    prompts = list(zc.requests(cfg, [30, 3, 17, 1, 22], 7).values())
    out = engine.generate(prompts, SamplingParams(temperature=0.0, max_new_tokens=12, ignore_eos=True))
    for prompt, tokens in zip(prompts, out):
        assert tokens == _greedy(cfg, w, prompt, 12)
    engine.runner.cache.check()
    assert not engine.runner.cache.requests


@pytest.mark.parametrize("dtype,tol", [("float32", TOL), ("bfloat16", 6e-2)])
def test_the_replay_program_serves_a_folder(tmp_path, dtype, tol):
    """As a folder comes: config.json without the bottleneck's size, which the file's tensors say."""
    from transformers_neuronx_amd.weights import write_random_model
    cfg = zc.config("a")
    folder = write_random_model(cfg, str(tmp_path / "m"), 12, dtype="bfloat16")
    raw = json.load(open(os.path.join(folder, "config.json")))
    for l in raw["layers"]:
        if l["type"] == "parallel":
            del l["mixer"]["right"]["rank"]
    json.dump(raw, open(os.path.join(folder, "config.json"), "w"))
    from safetensors.torch import save_file
    w = zc.weights(cfg, 12, torch.bfloat16)
    save_file({k: v.contiguous() for k, v in w.items()}, os.path.join(folder, "model.safetensors"))
    requests = zc.requests(cfg, [40, 9, 70, 3, 25], 13)
    expected = _expected(cfg, w, requests)
    steps, place = schedules.mixed(requests, max_tokens=192, page=64, seed=1, tail=6, max_live=4)
    out_dir = tmp_path / "out"
    proc = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", folder, "--dtype", dtype,
                           "--out", str(out_dir), "--max-tokens", "192"], input="\n".join(json.dumps(s) for s in steps),
                          capture_output=True, text=True, timeout=300)
    assert proc.returncode == 0, proc.stderr[-2000:]
    assert [l for l in proc.stdout.splitlines() if l.startswith("done")] == [f"done {s['step']}" for s in steps]
    over = 0
    for (step, row), (rid, pos) in place.items():
        got = np.fromfile(out_dir / f"{step}.f32", dtype="<f4").reshape(-1, cfg.vocab)[row]
        want = expected[rid][pos].numpy()
        over += np.abs(got - want).max() / np.abs(expected[rid].numpy()).max() >= tol
    assert over <= (0 if dtype == "float32" else 0.12 * len(place))


def test_the_command_line_serves_the_folder(tmp_path, capsys):
    """`opt_demo save --random --config` writes a folder of whatever architecture the config.json names, and
    `run --benchmark --profile` generates from it and times its kernels."""
    from transformers_neuronx_amd.opt import demo
    with open(tmp_path / "config.json", "w") as fp:
        json.dump(dict(zc.CASES["c"], init_std=0.3), fp)
    folder = str(tmp_path / "model")
    assert demo.main(["--amp", "bf16", "save", folder, "--random", "--config", str(tmp_path / "config.json")]) in (0, None)
    assert demo.main(["--amp", "bf16", "run", folder, "--batch_size", "2", "--n_positions", "40", "--prompt_len", "9",
                      "--top_k", "1", "--benchmark", "--profile", "--page_size", "16"]) in (0, None)
    text = capsys.readouterr().out
    assert "running ZudusunForSampling.from_pretrained" in text
    report = json.loads(next(line for line in text.splitlines() if line.startswith("{")))
    assert report["inferences"] == 10 and report["e2e_output_token_throughput"] > 0
    for kernel in ("tnx_channel_decays", "tnx_turn_heads", "tnx_memory_walk", "tnx_gated_norm", "tnx_qkv_prepare",
                   "tnx_attention_scored", "tnx_expert_mixture", "tnx_route", "tnx_row_activation"):
        assert kernel in text, kernel


@pytest.mark.parametrize("dtype,tol", [("float32", TOL), ("bfloat16", 6e-2)])
@pytest.mark.parametrize("seed", range(12))
def test_configurations_drawn_from_a_seed(seed, dtype, tol):
    cfg = zc.drawn(seed)
    w = zc.weights(cfg, seed, torch.bfloat16 if dtype == "bfloat16" else torch.float32)
    runner = zc.runner(cfg, w, dtype=dtype, kernels="hip", device=DEV, max_tokens=176)
    requests = zc.requests(cfg, [70, 33, 5, 1], seed)
    expected = _expected(cfg, w, requests)
    few = 0.12 if dtype == "bfloat16" else 0.0
    step_through(runner, expected, schedules.mixed(requests, max_tokens=176, page=16, seed=5, tail=8, max_live=3), tol, few)
    step_through(runner, expected, schedules.head_then_singles(requests, tail=20), tol, few)
