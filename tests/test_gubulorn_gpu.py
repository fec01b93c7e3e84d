"""Gubulorn on the GPU: every kernel of its parts alone against the plain implementation's function of the same
mechanism (float32 and bfloat16), the memories over steps cut anywhere in slots that others left full, token by token
and chunk by chunk, attention with a sink and a temperature and a key made to stand out far away, at page borders and
at the first token, the choice inside groups and experts without tensors, the engine under every way of cutting,
recorded decoding, generation through the entry point and the scheduler, the replay program and the command line."""
import json
import os
import subprocess
import sys
from types import SimpleNamespace

import numpy as np
import pytest
import torch

import plain_gubulorn as P
import gubulorn_cases as gc
import schedules
from test_gubulorn_cpu import TOL, _expected, _greedy, step_through
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


# steps of a request in slot 2 and, from the third step on, of another in slot 0: (request, from, to, slot). Runs of one
# token, of a few, just under and at the length from which they go by chunks here, at and around whole chunks, and long ones.
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
    # heads, query/key heads, n, v, taps
    (1, 1, 1, 1, 1), (4, 2, 16, 24, 4), (3, 1, 10, 7, 2), (2, 2, 64, 64, 4), (6, 3, 128, 40, 3), (2, 1, 256, 20, 4),
    (2, 2, 100, 16, 5), (5, 5, 33, 5, 7), (4, 1, 48, 64, 2)])
@pytest.mark.parametrize("delta", [True, False])
@pytest.mark.parametrize("by_chunks", [True, False])
def test_memories_across_steps_cut_anywhere(sizes, delta, by_chunks):
    """Convolution, unit vectors, decays, write weights and the recurrence over steps of 1, 2 and more tokens, two
    requests side by side in slots that former holders left full, every step of single tokens run twice (a recorded
    step is), against the whole sequence token by token. Decays from almost none to at once."""
    heads, groups, n, v, taps = sizes
    ops = _ops(torch.float32)
    ops.memory_by_chunks = by_chunks
    g = torch.Generator().manual_seed(4)
    qk, inner = groups * n, heads * v
    channels, before = 2 * qk + inner, 5
    conv = torch.randn(channels, taps, generator=g) * 0.6
    bias = None if delta else torch.randn(channels, generator=g) * 0.3
    a_log, dt_bias = torch.randn(heads, generator=g) * 1.5 - 1.0, torch.randn(heads, generator=g) * 1.5 - 1.5
    rate = -torch.exp(a_log)
    proj, want_u, want_o = {}, {}, {}
    share = [h // (heads // groups) for h in range(heads)]
    for r, t in LENGTHS.items():
        x = torch.randn(t, before + channels + 2 * heads + 3, generator=g) * 1.5
        proj[r] = x
        d = x.double()
        u = P.silu(P.short_conv(d[:, before:before + channels], conv.double(), None if bias is None else bias.double()))
        q, k, val = u[:, :qk].view(t, groups, n), u[:, qk:2 * qk].view(t, groups, n), u[:, 2 * qk:].view(t, heads, v)
        if delta:
            q, k = P.unit_vector(q) * n ** -0.5, P.unit_vector(k)
        want_u[r] = torch.cat([q.reshape(t, qk), k.reshape(t, qk), val.reshape(t, inner)], dim=1)
        at = before + channels
        dt = P.softplus(d[:, at:at + heads] + dt_bias.double())
        decay = rate.double() * dt
        if delta:
            o = P.delta_rule(q[:, share], k[:, share], val, decay, P.sigmoid(d[:, at + heads:at + 2 * heads]))
        else:
            o = P.state_space(val, k[:, share], q[:, share], decay, dt)
        want_o[r] = o.reshape(t, inner)
    memory = torch.full((3, 2, heads, v, n), 3.0, device=DEV)
    inputs = torch.full((3, taps, channels), -2.0, device=DEV) if taps > 1 else None
    for step in _steps():
        rows = torch.cat([proj[r][a:b] for r, a, b, _ in step]).to(DEV)
        ctx = _ctx([b - a for _, a, b, _ in step], [a for _, a, _, _ in step], [slot for _, _, _, slot in step],
                   planners=BY_CHUNKS)
        single = all(b - a == 1 for _, a, b, _ in step)
        for _ in range(2 if single else 1):
            u, decay, write = ops.memory_inputs(rows, before, conv.to(DEV), None if bias is None else bias.to(DEV), ctx, inputs,
                                                heads, before + channels, rate.to(DEV), dt_bias.to(DEV),
                                                write_at=before + channels + heads if delta else None,
                                                unit=(n, 2 * qk, qk, n ** -0.5) if delta else None)
            got = ops.linear_memory(u, 0, qk, 2 * qk, heads, groups, n, v, decay, write, ctx, memory, delta)
        at = 0
        for r, a, b, _ in step:
            _close(u[at:at + b - a], want_u[r][a:b], 1e-5, want_u[r].abs().max())
            _close(got[at:at + b - a], want_o[r][a:b], 3e-5, want_o[r].abs().max())
            at += b - a
    assert float(memory[1].min()) == 3.0 and float(memory[1].max()) == 3.0       # a slot of no one is not touched
    assert inputs is None or float(inputs[1].max()) == -2.0


@pytest.mark.parametrize("delta", [True, False])
def test_a_memory_that_remembers_hundreds_of_tokens_and_forgets_at_once(delta):
    """Head 0 hardly forgets: what the last token reads is what one token far back wrote, the keys between having
    nothing along it. Head 1 forgets everything at every token. Whole, by chunks and token by token, and decoded."""
    n, v, t = 64, 16, 400
    g = torch.Generator().manual_seed(2)
    k = torch.randn(t, n, generator=g)
    mark = torch.nn.functional.normalize(torch.randn(n, generator=g), dim=0)
    k = torch.nn.functional.normalize(k - (k @ mark)[:, None] * mark, dim=-1)
    k[3] = mark
    q = torch.nn.functional.normalize(torch.randn(t, n, generator=g), dim=-1) * 0.1
    q[-1] = mark
    val = torch.randn(t, 2, v, generator=g)
    log_decay = torch.stack([torch.full((t,), -1e-6), torch.full((t,), -60.0)], dim=1)
    write = torch.rand(t, 2, generator=g) * 0.5 + 0.5
    d = lambda x: x.double()
    qs, ks = d(q)[:, None].expand(t, 2, n), d(k)[:, None].expand(t, 2, n)
    want = (P.delta_rule(qs, ks, d(val), d(log_decay), d(write)) if delta
            else P.state_space(d(val), ks, qs, d(log_decay), d(write))).reshape(t, 2 * v)
    assert torch.allclose(want[-1, :v], d(write)[3, 0] * d(val)[3, 0] * math_exp(-1e-6 * (t - 4)), atol=1e-6)
    assert float(want[-1, v:].abs().max()) < 1e-20 or float((k[-1] * q[-1]).sum().abs()) > 1e-9
    u = torch.cat([q, k, val.reshape(t, 2 * v)], dim=1).to(DEV)
    for chunks, cuts in ((True, (0, t)), (False, (0, t)), (True, (0, 130, t - 1, t))):
        ops = _ops(torch.float32)
        ops.memory_by_chunks = chunks
        memory = torch.full((1, 2, 2, v, n), 9.0, device=DEV)
        out = []
        for a, b in zip(cuts[:-1], cuts[1:]):
            ctx = _ctx([b - a], [a], [0], planners=BY_CHUNKS)
            out.append(ops.linear_memory(u[a:b], 0, n, 2 * n, 2, 1, n, v, log_decay[a:b].to(DEV), write[a:b].to(DEV), ctx, memory, delta))
        got = torch.cat(out)
        _close(got, want, 1e-5)
        _close(got[-1, :v], want[-1, :v], 1e-5)


def math_exp(x):
    return torch.exp(torch.tensor(x, dtype=F64))


@pytest.mark.parametrize("name,dtype,tol", DTYPES)
@pytest.mark.parametrize("sizes", [
    # tokens, heads, elements a head, parts, the gate first
    (1, 1, 1, 1, True), (7, 4, 24, 4, False), (33, 6, 16, 2, True), (5, 3, 10, 5, True), (9, 32, 128, 8, True),
    (3, 5, 200, 5, False), (2, 70, 64, 1, True), (6, 4, 300, 4, False)])
def test_gate_norm_and_skip_behind_a_memory(name, dtype, tol, sizes):
    t, heads, v, parts, first = sizes
    width, eps = heads * v, 1e-3
    ops = _ops(dtype)
    g = torch.Generator().manual_seed(8)
    o, rows = torch.randn(t, width, generator=g) * 2, torch.randn(t, 2 * width + 7, generator=g) * 2
    weight, factors = torch.randn(width, generator=g), torch.randn(heads, generator=g)
    gate, x = rows[:, 5:5 + width], rows[:, 6 + width:6 + 2 * width]
    y, s = o.double(), P.silu(gate.double())
    if first:
        y = (y.view(t, heads, v) + factors.double()[None, :, None] * x.double().reshape(t, heads, v)).reshape(t, width) * s
    y = P.unit_rms(y.view(t, parts, -1), eps).reshape(t, width) * weight.double()
    want = y if first else y * s
    dev = rows.to(DEV)
    got = ops.gated_norm(o.to(DEV), dev[:, 5:5 + width], weight.to(DEV), eps, parts, first,
                         skip=(factors.to(DEV), dev[:, 6 + width:6 + 2 * width]) if first else None)
    _close(got, want, tol)


# ---------------------------------------------------------------- the sum, then the norm

@pytest.mark.parametrize("name,dtype,tol", DTYPES)
@pytest.mark.parametrize("width", [8, 50, 256, 1030, 2048, 4096, 8192, 9000])
def test_a_sum_with_a_factor_of_normed_results_and_its_norm(name, dtype, tol, width):
    ops = _ops(dtype)
    g = torch.Generator().manual_seed(width)
    t, eps, part_eps, alpha = 5, 1e-3, 1e-2, 2.3
    x, ya, yb = (torch.randn(t, width, generator=g) * s for s in (1.0, 5.0, 0.2))
    wa, wb, w = (torch.randn(width, generator=g) for _ in range(3))
    d = lambda z: z.double()
    for results, want in (
            ([(ya, None, None, 1.0)], alpha * d(x) + d(ya)),
            ([(ya, wa, part_eps, 0.5), (yb, wb, part_eps, 0.5)],
             alpha * d(x) + 0.5 * (P.unit_rms(d(ya), part_eps) * d(wa) + P.unit_rms(d(yb), part_eps) * d(wb))),
            ([(ya, None, None, -1.5), (yb, wb, part_eps, 3.0)], alpha * d(x) - 1.5 * d(ya) + 3.0 * P.unit_rms(d(yb), part_eps) * d(wb))):
        want = P.offset_norm(want, d(w), eps)
        dev = [(y.to(DEV), None if z is None else z.to(DEV), e, f) for y, z, e, f in results]
        h32, hc = ops.join_norm(x.to(DEV), alpha, dev, (1.0 + w).to(DEV), eps, dtype)
        _close(h32, want, 5e-6)
        _close(hc, want, tol)
        assert h32.dtype == torch.float32 and hc.dtype == dtype


def test_the_logits_scale_and_cap():
    ops = _ops(torch.float32)
    x = torch.randn(7, 333, generator=torch.Generator().manual_seed(0)) * 30
    for scale, cap in ((0.5, 15.0), (2.0, 0.0), (1.0, 3.0)):
        want = x.double() * scale
        want = cap * torch.tanh(want / cap) if cap else want
        _close(ops.scale_and_cap(x.clone().to(DEV), scale, cap), want, 1e-6)


# ---------------------------------------------------------------- attention with a temperature and a sink

@pytest.mark.parametrize("name,dtype,tol", DTYPES)
@pytest.mark.parametrize("coef,every", [(0.7, 1), (0.3, 7), (1.5, 16), (0.4, 1000)])
def test_queries_grow_by_the_temperature(name, dtype, tol, coef, every):
    ops = _ops(dtype)
    g = torch.Generator().manual_seed(3)
    heads, groups, n, v, d, ps, length = 6, 2, 20, 12, 32, 16, 60
    proj = torch.randn(length, heads * n + groups * (n + v), generator=g) * 2
    qw, kw = torch.randn(n, generator=g), torch.randn(n, generator=g)
    temp = P.query_temperature(range(length), coef, every)
    x = proj.double()
    q = P.unit_rms(x[:, :heads * n].view(length, heads, n), 1e-5) * qw.double() * 0.37 * temp[:, None, None]
    k = P.unit_rms(x[:, heads * n:heads * n + groups * n].view(length, groups, n), 1e-5) * kw.double()
    order = [5, 0, 3, 1]
    k_pages = torch.full((6, groups, ps, d), 7.0, dtype=dtype, device=DEV)
    v_pages = torch.full((6, groups, d, ps), 7.0, dtype=dtype, device=DEV)
    got = []
    for a, b in ((0, 1), (1, 3), (3, 20), (20, 21), (21, 60)):
        ctx = _ctx([b - a], [a], [0], {"g": [order]}, ps)
        got.append(ops.qkv_prepare(proj[a:b].to(DEV), heads, groups, n, v, d, qw.repeat(heads).to(DEV), kw.repeat(groups).to(DEV),
                                   1e-5, None, False, 0.37, None, None, ctx, ctx.groups["g"], k_pages, v_pages, per_head=True,
                                   temperature=(coef, every)))
    got = torch.cat(got).view(length, heads, d)
    _close(got[:, :, :n], q, tol)
    assert float(got[:, :, n:].abs().max()) == 0
    _close(torch.cat([k_pages[p] for p in order], dim=1)[:, :length, :n].permute(1, 0, 2), k, tol)      # keys have no temperature


@pytest.mark.parametrize("name,dtype,tol", [("float32", torch.float32, 4e-5), ("bfloat16", torch.bfloat16, 4e-2)])
@pytest.mark.parametrize("case", [
    # query heads, kv heads, key size, value size, cached size, length, the step's tokens, page, standout (back from the
    # last), the sinks' level: far above the other keys and below the one that stands out, above it, or nothing
    dict(h=4, g=2, n=16, v=16, d=16, length=300, run=1, ps=16, back=299, sink=0.0),      # the very first token, decoded alone
    dict(h=2, g=1, n=64, v=64, d=64, length=700, run=1, ps=16, back=697, sink=9.0),      # far away
    dict(h=2, g=1, n=64, v=64, d=64, length=700, run=300, ps=64, back=697, sink=3.0),    # far away, in a prompt (pipelined)
    dict(h=6, g=1, n=96, v=80, d=96, length=700, run=37, ps=64, back=640, sink=90.0),    # a page border; sinks that outweigh it
    dict(h=6, g=3, n=16, v=24, d=32, length=64, run=64, ps=16, back=63, sink=-60.0),     # a whole prompt; sinks of no weight
    dict(h=1, g=1, n=64, v=64, d=64, length=129, run=2, ps=64, back=1, sink=5.0),        # the token before: the last of a page
    dict(h=20, g=1, n=32, v=32, d=32, length=390, run=1, ps=64, back=200, sink=8.0),     # twenty heads on one key/value head
    dict(h=3, g=3, n=10, v=6, d=16, length=50, run=3, ps=16, back=0, sink=2.0),          # itself; heads filled up in the cache
    dict(h=8, g=2, n=128, v=128, d=128, length=280, run=200, ps=64, back=279, sink=70.0),  # several tiles; sinks that outweigh it
    dict(h=4, g=4, n=48, v=48, d=48, length=330, run=330, ps=64, back=300, sink=4.0),    # a set of tiles for each set of waves
    dict(h=4, g=2, n=160, v=144, d=160, length=300, run=140, ps=16, back=200, sink=3.0),
    dict(h=4, g=2, n=32, v=32, d=32, length=330, run=130, ps=48, back=329, sink=3.0),    # pages that are no power of two
])
@pytest.mark.parametrize("kernel", ["matrix unit", "shared out", "one set", "general"])
def test_attention_with_a_sink_finds_the_key_that_stands_out(name, dtype, tol, case, kernel):
    if kernel != "general" and dtype == torch.float32:
        pytest.skip("float32 has the one kernel")
    from transformers_neuronx_amd.kernels.attention_plan import attention_plan
    ops = _ops(dtype)
    ops.force_plain_attention = kernel == "general"
    ops.scored_decode_splits = 3 if kernel == "shared out" else 1
    ops.prefill_direct = {"one set": 2, "shared out": 3}.get(kernel, False)
    h, g, n, v, d, length, run, ps = (case[k] for k in ("h", "g", "n", "v", "d", "length", "run", "ps"))
    standout = length - 1 - case["back"]
    gen = torch.Generator().manual_seed(7)
    proj = torch.randn(length, h * n + g * (n + v) + h, generator=gen) * 0.3
    mark = torch.randn(n, generator=gen)
    mark = mark / mark.norm() * 6.0
    proj[standout, h * n:h * n + g * n] = mark.repeat(g)
    proj[length - 1, :h * n] = mark.repeat(h)
    proj[:, h * n + g * (n + v):] *= 6
    proj = proj.to(dtype).float()
    sink = torch.randn(h, generator=gen) + case["sink"]
    scale = 0.6
    x = proj.double()
    q = x[length - run:, :h * n].view(run, h, n)
    k = x[:, h * n:h * n + g * n].view(length, g, n).repeat_interleave(h // g, 1)
    val = x[:, h * n + g * n:h * n + g * (n + v)].view(length, g, v).repeat_interleave(h // g, 1)
    scores = torch.einsum("ihd,jhd->hij", q, k) * scale
    hidden = torch.arange(length)[None, :] > torch.arange(length - run, length)[:, None]
    scores = scores.masked_fill(hidden[None], -1e30)
    top = torch.maximum(scores.max(-1, keepdim=True).values, sink.double()[:, None, None])
    e = torch.exp(scores - top)
    prob = e / (e.sum(-1, keepdim=True) + torch.exp(sink.double()[:, None, None] - top))
    share = float(prob[:, -1, standout].max())
    assert (share < 1e-6) if case["sink"] > 50 else (share > 0.9), share
    want = torch.einsum("hij,jhd->ihd", prob, val) * P.sigmoid(x[length - run:, h * n + g * (n + v):])[:, :, None]
    blocks = -(-length // ps)
    order = torch.randperm(blocks + 3, generator=torch.Generator().manual_seed(1))[:blocks].tolist()
    k_pages = torch.full((blocks + 3, g, ps, d), 50.0, dtype=dtype, device=DEV)
    v_pages = torch.full((blocks + 3, g, d, ps), 50.0, dtype=dtype, device=DEV)
    for a, b in ((0, length - run), (length - run, length)):
        if b == a:
            continue
        ctx = _ctx([b - a], [a], [0], {"g": [order]}, ps, {"attention": attention_plan})
        rows = proj[a:b].to(DEV)
        qd = ops.qkv_prepare(rows, h, g, n, v, d, None, None, 0.0, None, False, scale, None, None, ctx, ctx.groups["g"], k_pages,
                             v_pages)
        got = ops.attention_scored(qd, h, g, d, ctx, ctx.groups["g"], k_pages, v_pages, gate=rows[:, h * n + g * (n + v):],
                                   value_size=v, gate_per_head=True, sink=sink.to(DEV))
    floor = 0.0 if case["sink"] <= 50 else 1e-9          # (sinks that outweigh everything leave almost nothing to compare)
    _close(got.view(run, h, d)[:, :, :v], want, tol, max(float(want.abs().max()), floor))


# ---------------------------------------------------------------- the mixture

@pytest.mark.parametrize("name,dtype,tol", DTYPES)
@pytest.mark.parametrize("sizes", [
    # tokens, experts, experts without tensors, a token's experts, groups, groups kept, width, inner size
    (1, 3, 1, 1, 2, 1, 64, 16), (37, 5, 3, 3, 4, 2, 96, 40), (130, 7, 0, 2, 1, 1, 192, 72), (9, 2, 4, 4, 3, 2, 50, 30),
    (300, 60, 12, 6, 8, 3, 128, 24), (900, 6, 2, 4, 4, 2, 128, 64), (700, 1, 1, 1, 1, 1, 64, 32), (40, 100, 50, 5, 75, 3, 32, 8)])
@pytest.mark.parametrize("forced", [None, "ours", "plain"])
def test_experts_chosen_inside_groups_and_experts_without_tensors(name, dtype, tol, sizes, forced):
    """`forced`: None, as the engine would (steps of many pairs an expert through the vendor library); "ours": the one
    launch of ours at any size; "plain": without the matrix unit."""
    from transformers_neuronx_amd.parts.feed_forward import ExpertMixture
    tokens, experts, identity, top, count, keep, width, inner = sizes
    if forced and (dtype == torch.float32 or (forced == "ours" and tokens < 100)):
        pytest.skip("the same path as unforced")
    ops = _ops(dtype)
    ops.expert_library_rows = 96 if forced is None else 0
    ops.expert_plain_products = forced == "plain"
    g = torch.Generator().manual_seed(5)
    part = ExpertMixture(width, experts, top, inner, "router", "e{}.", ("gate", "up", "down"), score="softmax",
                         weight_on="output", activation="silu", correction_name="correction", identity=identity,
                         groups=dict(count=count, keep=keep))
    w = {d.name: (torch.randn(d.shape, generator=g) * (2.0 / d.shape[-1] ** 0.5)).to(dtype) for d in part.param_decls("p.")}
    w["p.correction"] = torch.randn(experts + identity, generator=g) * 0.3 - 0.4       # many choice scores are negative
    part.load({k: v.to(DEV) for k, v in w.items()}, "p.", ops, dtype)
    h = torch.randn(tokens, width, generator=g).to(dtype)
    residual = torch.randn(tokens, width, generator=g)
    wide = P.widen(w)
    wide["p.correction"] = w["p.correction"].double()
    z = h.double() @ wide["p.router"].T
    chosen, weight = P.route(z, wide["p.correction"], top, count, keep)
    # only tokens whose choice float64 and float32 cannot see differently
    choice = torch.softmax(z, -1) + wide["p.correction"]
    moved = [P.route(z + torch.randn(z.shape, generator=torch.Generator().manual_seed(i), dtype=F64) * 1e-5,
                     wide["p.correction"], top, count, keep)[0] for i in range(3)]
    clear = torch.stack([(m == chosen).all(-1) for m in moved]).all(0)
    assert int(clear.sum()) >= max(1, tokens // 2)
    free, _ = P.route(z, wide["p.correction"], top, 1, 1)
    assert tokens < 30 or keep == count or chosen.tolist() != free.tolist()             # the groups matter here
    assert tokens < 100 or not identity or bool((chosen >= experts).any())
    got_chosen, got_weight = ops.route(ops.linear(h.to(DEV), part.w_router, None, out_f32=True)[:, :part.routed], top, "softmax", False,
                                       correction=part.correction, groups=(count, keep))
    assert got_chosen.cpu()[clear].tolist() == chosen[clear].tolist()
    _close(got_weight.cpu()[clear], weight[clear], 1e-5 if dtype == torch.float32 else 1e-2)
    mlp = dict(router=dict(experts=experts, top=top, groups=dict(count=count, keep=keep)), expert=dict(ff=inner))
    want = P.mixture(mlp, wide, "p.", h.double())
    got = part.forward(h.to(DEV), SimpleNamespace(length_bound=None), residual.to(DEV))
    _close(got.cpu()[clear], (residual.double() + want)[clear], tol)
    alone = part.forward(h.to(DEV), SimpleNamespace(length_bound=None), None)
    _close(alone.cpu()[clear], want[clear], tol)


@pytest.mark.parametrize("name,dtype,tol", DTYPES)
@pytest.mark.parametrize("rows", [1, 8, 40, 300])
def test_the_clamped_gated_feed_forward(name, dtype, tol, rows):
    from transformers_neuronx_amd.parts.feed_forward import GatedFeedForward
    ops = _ops(dtype)
    g = torch.Generator().manual_seed(rows)
    part = GatedFeedForward(128, 192, "clamped_swiglu", ("gate", "up", "down"), limit=0.7)
    w = {d.name: (torch.randn(d.shape, generator=g) * (1.5 / d.shape[1] ** 0.5)).to(dtype) for d in part.param_decls("p.")}
    part.load({k: v.to(DEV) for k, v in w.items()}, "p.", ops, dtype)
    h = torch.randn(rows, 128, generator=g).to(dtype)
    _close(part.forward(h.to(DEV), None, None), P.dense(dict(limit=0.7), P.widen(w), "p.", h.double()), tol)


# ---------------------------------------------------------------- the engine

@pytest.mark.parametrize("dtype,tol", [("float32", TOL), ("bfloat16", 6e-2)])
@pytest.mark.parametrize("name", sorted(gc.CASES))
def test_schedules_on_the_gpu(name, dtype, tol):
    cfg = gc.config(name)
    w = gc.weights(cfg, 3, torch.bfloat16 if dtype == "bfloat16" else torch.float32)
    runner = gc.runner(cfg, w, dtype=dtype, kernels="hip", device=DEV, max_tokens=208)
    requests = gc.requests(cfg, [70, 33, 5, 100, 1], 1)
    expected = _expected(cfg, w, requests)
    few = 0.15 if dtype == "bfloat16" else 0.0
    for made in (schedules.whole(requests), schedules.head_then_singles(requests, tail=12), schedules.portions(requests),
                 schedules.portions(requests, sizes=(2, 2, 3, 2, 16, 2, 15, 17, 2)),
                 schedules.mixed(requests, max_tokens=208, page=16, seed=5, tail=8, max_live=3),
                 schedules.only_last(schedules.mixed(requests, max_tokens=208, page=16, seed=6, tail=20, max_live=4))):
        step_through(runner, expected, made, tol, few)
    from transformers_neuronx_amd.kernels import hip
    assert {"linear_memory", "prepare", "experts", "gemm", "scored", "stream"} <= set(hip.loaded_libraries())


@pytest.mark.parametrize("dtype,tol", [("float32", TOL), ("bfloat16", 6e-2)])
def test_long_requests_under_every_way_of_cutting(dtype, tol):
    """Requests of several chunks and pages of 64."""
    cfg = gc.config("c")
    w = gc.weights(cfg, 5, torch.bfloat16 if dtype == "bfloat16" else torch.float32)
    runner = gc.runner(cfg, w, dtype=dtype, kernels="hip", device=DEV, max_tokens=1024, page_size=64)
    requests = gc.requests(cfg, [400, 129, 64, 250], 8)
    expected = _expected(cfg, w, requests)
    few = 0.15 if dtype == "bfloat16" else 0.0
    for made in (schedules.whole(requests), schedules.head_then_singles(requests, tail=20),
                 schedules.portions(requests, sizes=(70, 2, 63, 64, 65, 24, 23, 1, 128)),
                 schedules.mixed(requests, max_tokens=1024, page=64, seed=2, tail=10, max_live=4)):
        step_through(runner, expected, made, tol, few)


def test_the_stream_after_every_layer_on_the_gpu():
    from transformers_neuronx_amd import debug
    cfg = gc.config("c")
    w = gc.weights(cfg, 2)
    toks = gc.requests(cfg, [70], 0)["r0"]
    _, layers = P.forward(cfg.to_dict(), P.widen(w), toks, return_layers=True)
    runner = gc.runner(cfg, w, dtype="float32", kernels="hip", device=DEV)
    with debug.debug_context() as taps:
        runner.step([StepEntry("r0", toks, [])])
    for i, want in enumerate(layers):
        got = taps[f"call{i}.layer{i}"]
        assert float((got.double().cpu() - want).abs().max() / want.abs().max()) < 1e-5, i


@pytest.mark.parametrize("graphs", [True, False])
def test_long_decoding_recorded_and_not(graphs):
    """300 tokens one by one beside requests that join and leave: the batch size changes (a recorded step is made for
    each), pages and slots change hands."""
    cfg = gc.config("c")
    w = gc.weights(cfg, 8)
    runner = gc.runner(cfg, w, dtype="float32", kernels="hip", device=DEV, max_tokens=512, page_size=16, use_graphs=graphs)
    requests = gc.requests(cfg, [320, 90, 60], 9)
    expected = _expected(cfg, w, requests)
    a, b, c = requests["r0"], requests["r1"], requests["r2"]
    got = {"r0": [runner.step([StepEntry("r0", a[:20], list(range(20)))])], "r1": [], "r2": []}
    for i in range(20, 320):
        entries = [StepEntry("r0", [a[i]], [0])]
        if 50 <= i < 140:
            entries.append(StepEntry("r1", [b[i - 50]], [0]))
        if 200 <= i < 260:
            entries.append(StepEntry("r2", [c[i - 200]], [0]))
        out = runner.step(entries)
        for row, e in enumerate(entries):
            got[e.req].append(out[row:row + 1].clone())
        if i == 139:
            runner.finish("r1")
        if i == 259:
            runner.finish("r2")
    assert (runner.graph_replays > 0) == graphs
    for rid in requests:
        have = torch.cat(got[rid])
        assert float((have.double().cpu() - expected[rid]).abs().max() / expected[rid].abs().max()) < TOL, rid


def test_long_decoding_in_bfloat16_recorded():
    cfg = gc.config("c")
    w = gc.weights(cfg, 9, torch.bfloat16)
    runner = gc.runner(cfg, w, dtype="bfloat16", kernels="hip", device=DEV, max_tokens=1024, page_size=64)
    requests = gc.requests(cfg, [600, 200], 4)
    expected = _expected(cfg, w, requests)
    a, b = requests["r0"], requests["r1"]
    got = {"r0": [runner.step([StepEntry("r0", a[:300], list(range(300)))])], "r1": [runner.step([StepEntry("r1", b[:2], [0, 1])])]}
    for i in range(300, 600):
        entries = [StepEntry("r0", [a[i]], [0])] + ([StepEntry("r1", [b[i - 298]], [0])] if i - 298 < 200 else [])
        out = runner.step(entries)
        for row, e in enumerate(entries):
            got[e.req].append(out[row:row + 1].clone())
    assert runner.graph_replays > 0
    for rid in requests:
        have = torch.cat(got[rid])
        err = (have.double().cpu() - expected[rid]).abs().amax(-1) / expected[rid].abs().max()
        assert float((err > 6e-2).double().mean()) <= 0.15, rid


@pytest.mark.parametrize("amp,tol", [("f32", TOL), ("bf16", 6e-2)])
def test_generation_through_the_entry_point(tmp_path, amp, tol):
    from safetensors.torch import load_file
    from transformers_neuronx_amd import NeuronAutoModelForCausalLM
    from transformers_neuronx_amd.weights import write_random_model
    cfg = gc.config("a")
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
    cfg = gc.config("b")
    w = gc.weights(cfg, 6)
    ecfg = EngineConfig(dtype="float32", kernels="hip", device=DEV, page_size=16, max_tokens=96, max_num_seqs=3,
                        max_num_batched_tokens=24, chunk_size=9)
    engine = LLMEngine(build_runner(cfg, TensorDict(w), ecfg), ecfg)
    prompts = list(gc.requests(cfg, [30, 3, 17, 1, 22], 7).values())
    out = engine.generate(prompts, SamplingParams(temperature=0.0, max_new_tokens=12, ignore_eos=True))
    for prompt, tokens in zip(prompts, out):
        assert tokens == _greedy(cfg, w, prompt, 12)
    engine.runner.cache.check()
    assert not engine.runner.cache.requests


def test_the_replay_program_serves_a_folder(tmp_path):
    from transformers_neuronx_amd.weights import write_random_model
    cfg = gc.config("b")
    folder = write_random_model(cfg, str(tmp_path / "m"), 12, dtype="bfloat16")
    from safetensors.torch import load_file
    w = load_file(os.path.join(folder, "model.safetensors"))
    requests = gc.requests(cfg, [40, 9, 70, 3, 25], 13)
    expected = _expected(cfg, w, requests)
    steps, place = schedules.mixed(requests, max_tokens=192, page=64, seed=1, tail=6, max_live=4)
    out_dir = tmp_path / "out"
    proc = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", folder, "--dtype", "float32",
                           "--out", str(out_dir), "--max-tokens", "192"], input="\n".join(json.dumps(s) for s in steps),
                          capture_output=True, text=True, timeout=300)
    assert proc.returncode == 0, proc.stderr[-2000:]
    assert [l for l in proc.stdout.splitlines() if l.startswith("done")] == [f"done {s['step']}" for s in steps]
    for (step, row), (rid, pos) in place.items():
        got = np.fromfile(out_dir / f"{step}.f32", dtype="<f4").reshape(-1, cfg.vocab)[row]
        want = expected[rid][pos].numpy()
        assert np.abs(got - want).max() / np.abs(expected[rid].numpy()).max() < TOL


def test_the_command_line_serves_the_folder(tmp_path, capsys):
    """`opt_demo save --random --config` writes a folder of whatever architecture the config.json names, and
    `run --benchmark --profile` generates from it and times its kernels."""
    from transformers_neuronx_amd.opt import demo
    with open(tmp_path / "config.json", "w") as fp:
        json.dump(dict(gc.CASES["c"], init_std=0.3), fp)
    folder = str(tmp_path / "model")
    assert demo.main(["--amp", "bf16", "save", folder, "--random", "--config", str(tmp_path / "config.json")]) in (0, None)
    assert demo.main(["--amp", "bf16", "run", folder, "--batch_size", "2", "--n_positions", "40", "--prompt_len", "9",
                      "--top_k", "1", "--benchmark", "--profile", "--page_size", "16"]) in (0, None)
    text = capsys.readouterr().out
    assert "running GubulornForSampling.from_pretrained" in text
    report = json.loads(next(line for line in text.splitlines() if line.startswith("{")))
    assert report["inferences"] == 10 and report["e2e_output_token_throughput"] > 0
    for kernel in ("tnx_memory_inputs", "tnx_memory_walk", "tnx_gated_norm", "tnx_join_norm", "tnx_qkv_prepare",
                   "tnx_attention_scored", "tnx_expert_mixture", "tnx_route", "tnx_gated_activation", "tnx_scale_and_cap"):
        assert kernel in text, kernel


@pytest.mark.parametrize("dtype,tol", [("float32", TOL), ("bfloat16", 6e-2)])
@pytest.mark.parametrize("seed", range(12))
def test_configurations_drawn_from_a_seed(seed, dtype, tol):
    cfg = gc.drawn(seed)
    w = gc.weights(cfg, seed, torch.bfloat16 if dtype == "bfloat16" else torch.float32)
    runner = gc.runner(cfg, w, dtype=dtype, kernels="hip", device=DEV, max_tokens=176)
    requests = gc.requests(cfg, [70, 33, 5, 1], seed)
    expected = _expected(cfg, w, requests)
    few = 0.15 if dtype == "bfloat16" else 0.0
    step_through(runner, expected, schedules.mixed(requests, max_tokens=176, page=16, seed=5, tail=8, max_live=3), tol, few)
    step_through(runner, expected, schedules.head_then_singles(requests, tail=20), tol, few)
