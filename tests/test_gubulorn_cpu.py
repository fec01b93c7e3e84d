"""Gubulorn on the host: the plain implementation pinned by what its mechanisms must do, the configuration's reader,
and the engine (registry, loader, cache manager, step function, scheduler, entry point) on the torch rendition of the
kernels against the plain implementation, for configurations of the tests' own."""
import json
import math
import os

import pytest
import torch

import plain_gubulorn as P
import gubulorn_cases as gc
import schedules
from transformers_neuronx_amd.config import EngineConfig, read_config
from transformers_neuronx_amd.config.model_config import ConfigError
from transformers_neuronx_amd.engine import StepEntry
from transformers_neuronx_amd.engine.engine import LLMEngine
from transformers_neuronx_amd.gubulorn import GubulornConfig, gubulorn_spec
from transformers_neuronx_amd.sampling import SamplingParams
from transformers_neuronx_amd.weights import WeightsError, write_random_model

F64 = torch.float64
TOL = 6e-5       # float32 against the plain implementation's float64, as a share of the logits' range


# ---------------------------------------------------------------- the plain implementation, pinned

def test_plain_convolution_and_activations_in_plain_numbers():
    x = torch.tensor([[1.0], [2.0], [-3.0]], dtype=F64)
    w = torch.tensor([[10.0, 100.0, 1.0]], dtype=F64)            # the last column meets the current token
    assert P.short_conv(x, w)[:, 0].tolist() == [1.0, 2.0 + 100.0, -3.0 + 200.0 + 10.0]
    assert P.short_conv(x, w, torch.tensor([0.5], dtype=F64))[0, 0] == 1.5
    one = torch.tensor([[5.0]], dtype=F64)
    assert P.short_conv(x, one)[:, 0].tolist() == [5.0, 10.0, -15.0]
    assert abs(float(P.softplus(torch.tensor(0.0, dtype=F64))) - math.log(2)) < 1e-12
    assert float(P.softplus(torch.tensor(800.0, dtype=F64))) == 800.0
    assert float(P.unit_vector(torch.tensor([3.0, 4.0], dtype=F64)).norm()) == pytest.approx(1.0, abs=1e-6)
    assert P.offset_norm(torch.tensor([3.0, 3.0], dtype=F64), torch.tensor([0.0, 1.0], dtype=F64), 0.0).tolist() == [1.0, 2.0]


def test_plain_delta_rule_by_hand():
    # one head of one element: S <- d S; u = b (v - S k); S <- S + k u; o = S q, with the current write in the read-out
    one = lambda *v: torch.tensor(v, dtype=F64).view(-1, 1, 1)
    d, b = torch.log(torch.tensor([[0.5], [0.5]], dtype=F64)), torch.tensor([[1.0], [0.25]], dtype=F64)
    o = P.delta_rule(one(2.0, 3.0), one(1.0, 0.5), one(4.0, 8.0), d, b)
    s1 = 1.0 * 4.0
    s2 = 0.5 * s1
    s2 = s2 + 0.5 * 0.25 * (8.0 - s2 * 0.5)
    assert o.view(-1).tolist() == [2.0 * s1, 3.0 * s2]
    # a full write (beta 1, no decay) along a unit key replaces what the memory held along it and nothing else
    g = torch.Generator().manual_seed(0)
    k = torch.nn.functional.normalize(torch.randn(2, 1, 6, generator=g, dtype=F64), dim=-1)
    k[1] = torch.nn.functional.normalize(k[1] - (k[1] * k[0]).sum() * k[0], dim=-1)
    keys, q = torch.cat([k[0:1], k[1:2], k[0:1]]), torch.cat([k[0:1], k[1:2], k[1:2]])
    v = torch.randn(3, 1, 4, generator=g, dtype=F64)
    o = P.delta_rule(q, keys, v, torch.zeros(3, 1, dtype=F64), torch.ones(3, 1, dtype=F64))
    assert torch.allclose(o[0], v[0]) and torch.allclose(o[1], v[1]) and torch.allclose(o[2], v[1])
    assert torch.allclose(P.delta_rule(keys, keys, v, torch.zeros(3, 1, dtype=F64), torch.ones(3, 1, dtype=F64))[2], v[2])


def test_plain_state_space_by_hand():
    g = torch.Generator().manual_seed(1)
    x, b, c = (torch.randn(5, 1, n, generator=g, dtype=F64) for n in (3, 4, 4))
    dt = torch.rand(5, 1, generator=g, dtype=F64)
    y = P.state_space(x, b, c, -2.0 * dt, dt)
    # y_t = sum_j exp(-2 (dt_(j+1) + .. + dt_t)) dt_j (b_j . c_t) x_j
    for t in range(5):
        want = sum(math.exp(-2.0 * float(dt[j + 1:t + 1].sum())) * float(dt[j]) * float((b[j] * c[t]).sum()) * x[j, 0] for j in range(t + 1))
        assert torch.allclose(y[t, 0], want)


def test_plain_mamba_norms_after_the_gate_and_in_parts():
    m = dict(heads=2, vdim=4, state=3, groups=1, conv=2, norm_groups=2)
    cfg = GubulornConfig.from_dict(dict(gc.CASES["d"], width=10, layers=[
        gc.layer(gc.parallel((1, 1, 4, 4, 1.0, None), (2, 4, 3, 1, 2, 2)), None)]))
    w = P.widen(gc.weights(cfg, 3))
    p = "l0.mix.right."
    h = torch.randn(6, 10, dtype=F64)
    inner = 8
    same = dict(w, **{p + "o": torch.eye(inner, dtype=F64), p + "norm": torch.ones(inner, dtype=F64)})
    y = P.mamba2(m, same, p, h, 0.0)
    assert torch.allclose((y.view(6, 2, 4) ** 2).mean(-1), torch.ones(6, 2, dtype=F64))        # each part by its own root mean square
    # a gate row scaled: the part's direction changes, its size does not (the gate comes before the norm)
    scaled = dict(same, **{p + "in": w[p + "in"].clone()})
    scaled[p + "in"][0] *= 3.0
    z = P.mamba2(m, scaled, p, h, 0.0)
    assert torch.allclose((z.view(6, 2, 4) ** 2).mean(-1), torch.ones(6, 2, dtype=F64)) and not torch.allclose(y[:, :4], z[:, :4])
    assert torch.allclose(y[:, 4:], z[:, 4:])


def test_plain_attention_temperature_and_sink():
    t = P.query_temperature([0, 1, 2, 3, 6, 7], 0.5, 4)
    want = [1.0, 1.0, 1.0, 1.0 + 0.5 * math.log(2), 1.0 + 0.5 * math.log(2), 1.0 + 0.5 * math.log(3)]
    assert torch.allclose(t, torch.tensor(want, dtype=F64))
    s = torch.tensor([[[1.0, 9.0], [1.0, 1.0]]], dtype=F64)
    a = P.sink_weights(s, torch.tensor([1.0], dtype=F64))
    assert torch.allclose(a[0, 1], torch.full((2,), 1.0 / 3.0, dtype=F64)) and float(a[0, 0, 1]) == 0 and float(a[0, 0, 0]) == 0.5
    # the first token's result: its own value times its share beside the sink, through its head's gate
    cfg = gc.config("a")
    m, w, p = cfg.layers[1]["mixer"]["left"], P.widen(gc.weights(cfg, 0)), "l1.mix.left."
    h = torch.randn(4, cfg.width, dtype=F64)
    q = P.unit_rms((h[0] @ w[p + "q"].T).view(6, 16), cfg.eps) * w[p + "q.norm"]
    k = P.unit_rms((h[0] @ w[p + "k"].T).view(2, 16), cfg.eps) * w[p + "k.norm"]
    score = (q * k.repeat_interleave(3, 0)).sum(-1) * m["scale"]
    share = 1.0 / (1.0 + torch.exp(w[p + "sink"] - score)) * torch.sigmoid(h[0] @ w[p + "g"].T)
    val = (h[0] @ w[p + "v"].T).view(2, 32).repeat_interleave(3, 0)
    assert torch.allclose(P.attention(m, w, p, h, cfg.eps)[0], (val * share[:, None]).reshape(-1) @ w[p + "o"].T)


def test_plain_router_chooses_inside_the_best_groups():
    z = torch.log(torch.tensor([[0.30, 0.05, 0.20, 0.21, 0.04, 0.20]], dtype=F64))
    none = torch.zeros(6, dtype=F64)
    chosen, weight = P.route(z, none, 2, 3, 1)                     # groups (0, 1), (2, 3), (4, 5): the first is best
    assert chosen.tolist() == [[0, 1]] and torch.allclose(weight, torch.tensor([[0.30, 0.05]], dtype=F64))
    assert P.route(z, none, 2, 3, 2)[0].tolist() == [[0, 3]]
    assert P.route(z, none, 3, 1, 1)[0].tolist() == [[0, 3, 2]]
    # the correction decides groups and experts, also where it makes every score negative, and is not in the weights
    corr = torch.tensor([-9.0, -1.0, -2.0, -3.0, -4.0, -5.0], dtype=F64)
    chosen, weight = P.route(z, corr, 2, 3, 1)
    assert chosen.tolist() == [[1, 0]] and torch.allclose(weight, torch.tensor([[0.05, 0.30]], dtype=F64))
    # an expert without tensors hands its input through, times its weight
    mlp = dict(router=dict(experts=1, identity=1, top=1, groups=dict(count=1, keep=1)), expert=dict(ff=2))
    h = torch.randn(1, 3, dtype=F64)
    w = {"p.router": torch.zeros(2, 3, dtype=F64), "p.correction": torch.tensor([0.0, 1.0], dtype=F64)}
    assert torch.allclose(P.mixture(mlp, w, "p.", h), 0.5 * h)


def test_plain_clamped_feed_forward_in_plain_numbers():
    w = {"gate": torch.tensor([[1.0]], dtype=F64), "up": torch.tensor([[-1.0]], dtype=F64), "down": torch.tensor([[2.0]], dtype=F64)}
    got = P.dense(dict(limit=1.0), w, "", torch.tensor([[3.0], [0.5], [-4.0]], dtype=F64))[:, 0].tolist()
    sig = lambda x: 1.0 / (1.0 + math.exp(-1.702 * x))
    want = [2 * (1.0 * sig(1.0) * (-1.0 + 1)), 2 * (0.5 * sig(0.5) * (-0.5 + 1)), 2 * (-4.0 * sig(-4.0) * (1.0 + 1))]
    assert all(abs(a - b) < 1e-12 for a, b in zip(got, want))


def test_plain_model_norms_after_the_sums():
    cfg = gc.config("d")
    raw, w = cfg.to_dict(), P.widen(gc.weights(cfg, 1))
    logits, layers = P.forward(raw, w, [3, 5, 7], return_layers=True)
    for i, x in enumerate(layers):
        assert torch.allclose(((x / (1.0 + w[f"l{i}.norm2"])) ** 2).mean(-1), torch.ones(3, dtype=F64), atol=2e-2)
    capped = dict(raw, logit_scale=2.0, logit_softcap=0.5)
    assert torch.allclose(P.forward(capped, w, [3, 5, 7]), 0.5 * torch.tanh(4.0 * logits))


# ---------------------------------------------------------------- configuration and weights

def test_config_reads_the_nested_keys_and_names_the_one_at_fault(tmp_path):
    cfg = gc.config("a")
    assert (cfg.eps, cfg.postln_alpha, cfg.logit_scale, cfg.logit_softcap, len(cfg.layers)) == (1e-4, 2.6, 0.75, 9.0, 4)
    assert gc.config("b").logit_softcap is None and gc.config("b").logit_scale == 1.0
    spec = gubulorn_spec(cfg)
    assert [l.mixer.kind for l in spec.layers] == ["gated_delta", "side_by_side", "gated_delta", "side_by_side"]
    assert [l.feed_forward.kind for l in spec.layers] == ["mixture", "gated", "none", "mixture"]
    assert spec.unread == ("l2.norm2",)
    folder = write_random_model(cfg, str(tmp_path / "m"), 0, dtype="float32")
    arch, read = read_config(folder)
    assert arch.name == "Gubulorn" and read.layers == cfg.layers and read.to_dict() == dict(cfg.to_dict(), torch_dtype="float32")
    raw = json.load(open(os.path.join(folder, "config.json")))

    def broken(change):
        r = json.loads(json.dumps(raw))
        change(r)
        return r
    for change, text in ((lambda r: r["norm"].pop("eps"), "norm.eps"),
                         (lambda r: r["layers"][2].update(type="other"), r"layers\[2\].type"),
                         (lambda r: r["layers"][0]["mixer"].pop("conv"), r"layers\[0\].mixer.conv"),
                         (lambda r: r["layers"][0]["mixer"].update(kv_heads=3), r"layers\[0\].mixer.heads"),
                         (lambda r: r["layers"][1]["mixer"].pop("left"), r"layers\[1\].mixer.left.heads"),
                         (lambda r: r["layers"][1].pop("mixer"), r"layers\[1\].mixer"),
                         (lambda r: r["layers"][1]["mixer"]["left"].pop("scale"), r"mixer.left.scale"),
                         (lambda r: r["layers"][1]["mixer"]["left"]["q_temp"].update(every=0), r"q_temp.every"),
                         (lambda r: r["layers"][1]["mixer"]["right"].update(groups=3), r"mixer.right.heads"),
                         (lambda r: r["layers"][1]["mixer"]["right"].update(norm_groups=5), r"mixer.right.norm_groups"),
                         (lambda r: r["layers"][1]["mixer"]["right"].pop("state"), r"mixer.right.state"),
                         (lambda r: r["layers"][1]["mlp"].pop("limit"), r"layers\[1\].mlp.limit"),
                         (lambda r: r["layers"][0]["mlp"]["router"].update(top=5), "router.top"),
                         (lambda r: r["layers"][0]["mlp"]["router"]["groups"].update(count=3), "router.groups"),
                         (lambda r: r["layers"][0]["mlp"]["router"]["groups"].update(keep=5), "router.groups"),
                         (lambda r: r["layers"][0]["mlp"]["router"].update(identity=-1), "router.identity"),
                         (lambda r: r["layers"][0]["mlp"]["expert"].pop("ff"), "expert.ff"),
                         (lambda r: r["layers"][0]["mlp"].update(kind="other"), r"layers\[0\].mlp.kind"),
                         (lambda r: r.update(logit_softcap=-1.0), "logit_softcap"),
                         (lambda r: r.pop("postln_alpha"), "postln_alpha"),
                         (lambda r: r.pop("width"), "width")):
        with pytest.raises(ConfigError, match=text):
            GubulornConfig.from_dict(broken(change))


def test_the_loader_names_what_is_missing_and_passes_over_an_unread_norm(tmp_path):
    from safetensors.torch import load_file, save_file
    from transformers_neuronx_amd.engine.factory import runner_from_folder
    cfg = gc.config("a")
    folder = write_random_model(cfg, str(tmp_path / "m"), 0, dtype="float32")
    t = load_file(os.path.join(folder, "model.safetensors"))
    shapes = {"embed.norm": (96,), "l0.norm2": (96,), "l0.mix.q": (32, 96), "l0.mix.v": (96, 96), "l0.mix.v.conv": (96, 4),
              "l0.mix.b": (4, 96), "l0.mix.A_log": (4,), "l0.mix.norm": (24,), "l0.mix.g": (96, 96), "l0.mlp.router": (8, 96),
              "l0.mlp.correction": (8,), "l0.mlp.e4.down": (96, 40), "l1.mix.left.k": (32, 96), "l1.mix.left.v": (64, 96),
              "l1.mix.left.q.norm": (16,), "l1.mix.left.sink": (6,), "l1.mix.left.g": (6, 96), "l1.mix.left.o": (96, 192),
              "l1.mix.right.in": (32 + 32 + 48 + 48 + 4, 96), "l1.mix.right.conv": (128, 3), "l1.mix.right.conv.b": (128,),
              "l1.mix.right.D": (4,), "l1.mix.right.norm": (32,), "l1.mix.left.out": (96,), "l1.mlp.gate": (72, 96)}
    for name, shape in shapes.items():
        assert tuple(t[name].shape) == shape, name
    assert "l2.norm2" not in t and "l0.mlp.e5.up" not in t
    ecfg = EngineConfig(dtype="float32", kernels="reference", device="cpu", max_tokens=64)
    save_file(dict(t, **{"l2.norm2": torch.zeros(96)}), os.path.join(folder, "model.safetensors"))
    runner_from_folder(folder, ecfg)
    bad = dict(t)
    del bad["l3.mix.right.dt_bias"]
    bad["l0.mix.sink"] = torch.zeros(4)
    save_file(bad, os.path.join(folder, "model.safetensors"))
    with pytest.raises(WeightsError) as e:
        runner_from_folder(folder, ecfg)
    assert "l3.mix.right.dt_bias" in str(e.value) and "l0.mix.sink" in str(e.value)


# ---------------------------------------------------------------- the engine on the host

def _expected(cfg, w, requests):
    raw, wide = cfg.to_dict(), P.widen(w)
    return {rid: P.forward(raw, wide, toks) for rid, toks in requests.items()}


def step_through(runner, expected, made, tol, few_over=0.0):
    """`few_over`: the share of positions that may lie over `tol`, by any distance: in bfloat16 a rounding of the
    router's input changes which expert a token takes where two scores are close, and that token's result is
    another expert's. float32 allows none."""
    steps, place = made
    over, seen = [], 0
    for rec in steps:
        logits = runner.step([StepEntry(e["id"], e["tokens"], e["want"]) for e in rec["entries"]])
        for row in range(0 if logits is None else logits.shape[0]):
            rid, pos = place[(rec["step"], row)]
            want = expected[rid][pos]
            err = float((logits[row].double().cpu() - want).abs().max() / expected[rid].abs().max())
            seen += 1
            if not err < tol:
                over.append((rec["step"], rid, pos, err))
            assert few_over or err < tol, (rec["step"], rid, pos, err)
        for rid in rec["end"]:
            runner.finish(rid)
        runner.cache.check()
    assert len(over) <= few_over * seen, over[:5]
    assert not runner.cache.requests


def test_the_stream_after_every_layer():
    from transformers_neuronx_amd import debug
    cfg = gc.config("a")
    w = gc.weights(cfg, 2)
    toks = gc.requests(cfg, [19], 0)["r0"]
    _, layers = P.forward(cfg.to_dict(), P.widen(w), toks, return_layers=True)
    runner = gc.runner(cfg, w)
    with debug.debug_context() as taps:
        runner.step([StepEntry("r0", toks, [])])
    for i, want in enumerate(layers):
        got = taps[f"call{i}.layer{i}"]
        assert float((got.double() - want).abs().max() / want.abs().max()) < 1e-5, i


@pytest.mark.parametrize("name", sorted(gc.CASES))
def test_schedules_on_the_host(name):
    cfg = gc.config(name)
    w = gc.weights(cfg, 3)
    runner = gc.runner(cfg, w, max_tokens=208)
    requests = gc.requests(cfg, [70, 33, 5, 100, 1], 1)
    expected = _expected(cfg, w, requests)
    for made in (schedules.whole(requests), schedules.head_then_singles(requests, tail=12), schedules.portions(requests),
                 schedules.portions(requests, sizes=(2, 2, 3, 2, 16, 2, 15, 17, 2)),
                 schedules.mixed(requests, max_tokens=208, page=16, seed=5, tail=8, max_live=3),
                 schedules.only_last(schedules.mixed(requests, max_tokens=208, page=16, seed=6, tail=20, max_live=4))):
        step_through(runner, expected, made, TOL)


def test_pages_and_slots_that_are_used_again():
    """One request at a time in a pool that holds one: every request gets the pages and the slot the one before left
    full."""
    cfg = gc.config("b")
    w = gc.weights(cfg, 4)
    runner = gc.runner(cfg, w, max_tokens=48, max_seqs=1)
    requests = gc.requests(cfg, [37, 20, 3, 45], 2)
    expected = _expected(cfg, w, requests)
    for rid, toks in requests.items():
        assert all(g.pool.num_free == g.pool.num_pages for g in runner.cache.groups.values())
        got = runner.step([StepEntry(rid, toks[:2], [0, 1])])
        got = torch.cat([got, runner.step([StepEntry(rid, toks[2:], list(range(len(toks) - 2)))])])
        assert float((got.double() - expected[rid]).abs().max() / expected[rid].abs().max()) < TOL
        runner.finish(rid)


def test_long_decoding_on_the_host():
    cfg = gc.config("d")
    w = gc.weights(cfg, 5)
    runner = gc.runner(cfg, w, max_tokens=160, max_seqs=2)
    toks = gc.requests(cfg, [150], 3)["r0"]
    expected = _expected(cfg, w, {"r0": toks})["r0"]
    got = [runner.step([StepEntry("r0", toks[:3], list(range(3)))])]
    for t in toks[3:]:
        got.append(runner.step([StepEntry("r0", [t], [0])]))
    got = torch.cat(got)
    assert float((got.double() - expected).abs().max() / expected.abs().max()) < TOL


def test_two_mixers_side_by_side_with_normed_results_under_another_arrangement():
    """The mixer's own sum (`forward`) is what the arrangement makes of its results: norms, factors, the residual."""
    from transformers_neuronx_amd.engine.batch import build_context
    from transformers_neuronx_amd.kernels import make_ops
    from transformers_neuronx_amd.cache.manager import CacheManager
    from transformers_neuronx_amd.parts.base import MIXERS
    cfg = gc.config("a")
    spec = gubulorn_spec(cfg).layers[1].mixer
    mixer = MIXERS.build(spec)
    ops = make_ops("reference", torch.float32, "cpu")
    w = gc.weights(cfg, 0)
    mixer.load(w, "l1.mix.", ops, torch.float32)
    h, residual = torch.randn(7, cfg.width), torch.randn(7, cfg.width)
    m = cfg.layers[1]["mixer"]
    want = residual.double() + P.parallel(m, P.widen(w), "l1.mix.", h.double(), cfg.eps)
    runner = gc.runner(cfg, w)
    packed = runner.prepare([StepEntry("r", [0] * 7, [])])
    from transformers_neuronx_amd.engine.batch import context_from
    ctx = context_from(packed, torch.from_numpy(packed.flat))
    cid = runner.model.schedule[1][1]
    got = mixer.forward(h, ctx, runner.cache.caches[cid], residual)
    assert torch.allclose(got.double(), want, atol=2e-5)
    alone = mixer.forward(h, ctx, runner.cache.caches[cid], None)
    assert torch.allclose(alone.double(), want - residual.double(), atol=2e-5)


def _greedy(cfg, w, prompt, new):
    raw, wide = cfg.to_dict(), P.widen(w)
    toks = list(prompt)
    for _ in range(new):
        toks.append(int(P.forward(raw, wide, toks)[-1].argmax()))
    return toks[len(prompt):]


@pytest.mark.parametrize("run_ahead", [False, True])
def test_greedy_generation_through_the_scheduler(run_ahead):
    cfg = gc.config("b")
    w = gc.weights(cfg, 6)
    ecfg = EngineConfig(dtype="float32", kernels="reference", device="cpu", page_size=16, max_tokens=96, max_num_seqs=3,
                        max_num_batched_tokens=24, chunk_size=9, run_ahead=run_ahead)
    from transformers_neuronx_amd.engine.factory import build_runner
    from transformers_neuronx_amd.weights.loader import TensorDict
    engine = LLMEngine(build_runner(cfg, TensorDict(w), ecfg), ecfg)
    prompts = list(gc.requests(cfg, [30, 3, 17, 1, 22], 7).values())
    out = engine.generate(prompts, SamplingParams(temperature=0.0, max_new_tokens=12, ignore_eos=True))
    for prompt, tokens in zip(prompts, out):
        assert tokens == _greedy(cfg, w, prompt, 12)
    engine.runner.cache.check()
    assert not engine.runner.cache.requests


def test_generation_through_the_entry_point_on_the_host(tmp_path):
    from safetensors.torch import load_file
    from transformers_neuronx_amd import NeuronAutoModelForCausalLM
    from transformers_neuronx_amd.gubulorn.model import GubulornForSampling
    cfg = gc.config("a")
    folder = write_random_model(cfg, str(tmp_path / "m"), 11, dtype="float32")
    w = load_file(os.path.join(folder, "model.safetensors"))
    model = NeuronAutoModelForCausalLM.from_pretrained(folder, batch_size=2, amp="f32", n_positions=64, page_size=16,
                                                       kernels="reference", device="cpu")
    assert type(model) is GubulornForSampling
    model.to_neuron()
    ids = torch.tensor([[5, 200, 17, 3], [9, 9, 100, 42]])
    out = model.sample(ids, sequence_length=14, top_k=1)
    for row in range(2):
        assert out[row, 4:].tolist() == _greedy(cfg, w, ids[row].tolist(), 10)


@pytest.mark.parametrize("seed", range(10))
def test_configurations_drawn_from_a_seed_on_the_host(seed):
    cfg = gc.drawn(seed)
    w = gc.weights(cfg, seed)
    runner = gc.runner(cfg, w, max_tokens=176)
    requests = gc.requests(cfg, [70, 33, 5, 1], seed)
    step_through(runner, _expected(cfg, w, requests), schedules.mixed(requests, max_tokens=176, page=16, seed=5, tail=8, max_live=3), TOL)


def test_the_plan_of_a_step_names_the_chunks_of_its_long_runs():
    import numpy as np
    from transformers_neuronx_amd.kernels.memory_plan import MEMORY_CHUNK, MEMORY_LONG, memory_plan
    lens = np.array([1, MEMORY_LONG - 1, MEMORY_LONG, 2 * MEMORY_CHUNK, 1, 2 * MEMORY_CHUNK + 1])
    plan, host = memory_plan(lens, np.zeros(6, dtype=np.int64), 16)
    assert host == {"memory_walk_most": MEMORY_LONG - 1} and MEMORY_CHUNK < MEMORY_LONG <= 2 * MEMORY_CHUNK
    assert plan["memory_long_run"].tolist() == [2, 3, 5] and plan["memory_long_first"].tolist() == [0, 2, 4]
    assert plan["memory_chunk_run"].tolist() == [2, 2, 3, 3, 5, 5, 5]
    assert plan["memory_chunk_begin"].tolist() == [0, MEMORY_CHUNK] * 2 + [0, MEMORY_CHUNK, 2 * MEMORY_CHUNK]
    few, _ = memory_plan(lens, np.zeros(6, dtype=np.int64), 16, least=2)
    assert few["memory_long_run"].tolist() == [1, 2, 3, 5]
    none, _ = memory_plan(np.array([1, 2]), np.zeros(2), 16)
    assert all(v.size == 0 and v.dtype == np.int32 for v in none.values())
