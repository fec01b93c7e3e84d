"""Zudusun on the host: the plain implementation pinned by what its mechanisms must do, the configuration's reader, and
the engine (registry, loader, cache manager, step function, scheduler, entry point) on the torch rendition of the
kernels against the plain implementation, for configurations of the tests' own."""
import json
import math
import os

import pytest
import torch

import plain_zudusun as P
import schedules
import zudusun_cases as zc
from transformers_neuronx_amd.config import EngineConfig, read_config
from transformers_neuronx_amd.config.model_config import ConfigError
from transformers_neuronx_amd.engine import StepEntry
from transformers_neuronx_amd.engine.engine import LLMEngine
from transformers_neuronx_amd.sampling import SamplingParams
from transformers_neuronx_amd.weights import WeightsError, write_random_model
from transformers_neuronx_amd.zudusun import ZudusunConfig, zudusun_spec

F64 = torch.float64
TOL = 3e-5       # float32 against the plain implementation's float64, as a share of the logits' range


# ---------------------------------------------------------------- the plain implementation, pinned

def test_plain_norm_and_activations_in_plain_numbers():
    x = torch.tensor([[1.0, 3.0, 5.0, 7.0]], dtype=F64)          # mean 4, mean squared deviation 5
    w = torch.tensor([1.0, 2.0, 3.0, 4.0], dtype=F64)
    assert torch.allclose(P.centred_norm(x, w, 4.0), torch.tensor([[-1.0, -2.0 / 3, 1.0, 4.0]], dtype=F64))
    assert P.unit_rms(torch.tensor([3.0, 4.0], dtype=F64), 12.5).tolist() == [0.6, 0.8]
    assert P.squared_relu(torch.tensor([-2.0, 3.0])).tolist() == [0.0, 9.0]
    assert abs(float(P.log_sigmoid(torch.tensor(0.0, dtype=F64))) + math.log(2)) < 1e-12
    assert float(P.log_sigmoid(torch.tensor(-800.0, dtype=F64))) == -800.0


def test_plain_turns_are_rotations_of_their_pairs():
    g = torch.Generator().manual_seed(0)
    x, at = torch.randn(5, 2, 10, generator=g, dtype=F64), torch.tensor([0, 1, 7, 100, 3])
    for turn, pairs in ((P.turn_neighbours, [(0, 1), (2, 3), (4, 5)]), (P.turn_halves, [(0, 3), (1, 4), (2, 5)])):
        y = turn(x, at, 50.0, 6)
        assert torch.equal(y[:, :, 6:], x[:, :, 6:]) and torch.equal(y[0], x[0])
        for i, (a, b) in enumerate(pairs):
            z = torch.complex(x[:, :, a], x[:, :, b]) * torch.exp(1j * at[:, None] * 50.0 ** (-2.0 * i / 6))
            assert torch.allclose(y[:, :, a], z.real) and torch.allclose(y[:, :, b], z.imag)


def test_plain_attention_by_hand():
    # equal scores of 0: with the one in the denominator a query that sees m keys gives each 1 / (m + 1)
    q, k = torch.zeros(4, 2, 3, dtype=F64), torch.randn(4, 1, 3, dtype=F64)
    v = torch.tensor([1.0, 10.0, 100.0, 1000.0], dtype=F64).view(4, 1, 1)
    assert torch.allclose(P.attend(q, k, v, 0.5, 2, True)[:, 1, 0], torch.tensor([1 / 2, 11 / 3, 110 / 3, 1100 / 3], dtype=F64))
    assert torch.allclose(P.attend(q, k, v, 0.5, None, False)[:, 0, 0], torch.tensor([1, 5.5, 37, 277.75], dtype=F64))
    # large and very negative scores
    big = P.attend(torch.ones(1, 1, 1, dtype=F64), torch.tensor([[[900.0]]], dtype=F64), v[:1], 1.0, 5, True)
    assert float(big) == 1.0
    small = P.attend(torch.ones(1, 1, 1, dtype=F64), torch.tensor([[[-900.0]]], dtype=F64), v[:1], 1.0, 5, True)
    assert float(small) == 0.0
    # query heads share key/value heads in order
    q = torch.randn(3, 4, 2, dtype=F64)
    k, v = torch.randn(3, 2, 2, dtype=F64), torch.randn(3, 2, 5, dtype=F64)
    both = P.attend(q, k, v, 1.0)
    assert torch.allclose(both[:, 2:], P.attend(q[:, 2:], k[:, 1:], v[:, 1:], 1.0))


def test_plain_memory_is_a_sum_over_the_past():
    g = torch.Generator().manual_seed(1)
    q, k = torch.randn(6, 2, 3, generator=g, dtype=F64), torch.randn(6, 2, 3, generator=g, dtype=F64)
    v, ld = torch.randn(6, 2, 4, generator=g, dtype=F64), -torch.rand(6, 2, 3, generator=g, dtype=F64)
    o = P.decaying_memory(q, k, v, ld)
    for t in range(6):
        want = sum((q[t] * k[j] * torch.exp(ld[j + 1:t + 1].sum(0))).sum(-1)[:, None] * v[j] for j in range(t + 1))
        assert torch.allclose(o[t], want)


def test_plain_gated_linear_side_in_plain_numbers():
    # one head of one channel, one value: S_1 = k v; S_2 = alpha S_1 + k v; o = q S; the norm leaves sign(o) * weight
    m = dict(heads=1, dim=1, vdim=2, tau=4.0)
    one = lambda *x: torch.tensor(x, dtype=F64).view(-1, 1)
    w = {"q": one(2.0), "k": one(1.0), "v": one(1.0, -0.5), "g": one(1.0, 1.0), "a1": one(3.0), "a2": one(0.5),
         "a2.b": torch.tensor([0.25], dtype=F64), "norm": torch.tensor([1.0, 2.0], dtype=F64), "o": torch.eye(2, dtype=F64)}
    h = one(1.0, 2.0)
    s = torch.tensor([1.0, -0.5], dtype=F64)
    s = s * (1 / (1 + math.exp(-(3.0 * 2.0 * 0.5 + 0.25)))) ** 0.25 + 2.0 * torch.tensor([2.0, -1.0], dtype=F64)
    want = P.unit_rms(4.0 * s, 0.1) * w["norm"] * P.silu(torch.tensor(2.0, dtype=F64))
    assert torch.allclose(P.gated_linear_side(m, w, "", h, 0.1)[1], want)


def test_plain_retention_decays_by_its_list_and_scales_its_keys():
    m = dict(heads=2, dim=4, vdim=1, decay=[0.5, 1.0], rot=dict(base=10.0, dims=0))
    g = torch.Generator().manual_seed(2)
    w = {n: torch.randn(8, 3, generator=g, dtype=F64) for n in ("q", "k")}
    w["v"], w["g"] = (torch.randn(2, 3, generator=g, dtype=F64) for _ in range(2))
    w["o"] = torch.eye(2, dtype=F64)
    h = torch.randn(3, 3, generator=g, dtype=F64)
    q, k, v = (h @ w["q"].T).view(3, 2, 4), (h @ w["k"].T).view(3, 2, 4), h @ w["v"].T
    o = torch.stack([sum(torch.tensor([0.5, 1.0], dtype=F64) ** (2 - j) * (q[2] * k[j]).sum(-1) / 2.0 * v[j] for j in range(3))])
    want = o / torch.sqrt(o * o + 0.01) * P.silu(h[2] @ w["g"].T)
    assert torch.allclose(P.retention(m, w, "", h, 0.01)[2], want[0])


def test_plain_router_and_shared_expert():
    z = torch.tensor([[1.0, 3.0, 3.0, 2.0]], dtype=F64)
    chosen, weight = P.route(z, 3)
    e = math.exp(-1.0)
    assert chosen.tolist() == [[1, 2, 3]] and torch.allclose(weight, torch.tensor([[1.0, 1.0, e]], dtype=F64) / (2 + e))
    # one expert a token: weight 1, whatever its logit; the bias decides; the shared expert times its gate
    mlp = dict(router=dict(experts=2, top=1), shared=dict(ff=1))
    w = {"router": torch.tensor([[1.0], [0.5]], dtype=F64), "router.b": torch.tensor([0.0, 0.6], dtype=F64),
         "shared.sg": torch.tensor([[2.0]], dtype=F64)}
    for e, s in (("e0.", 10.0), ("e1.", 100.0), ("shared.", 1000.0)):
        w[e + "up"], w[e + "down"] = torch.tensor([[1.0]], dtype=F64), torch.tensor([[s]], dtype=F64)
    got = P.mixture(mlp, w, "", torch.tensor([[1.0], [2.0], [-3.0]], dtype=F64))[:, 0].tolist()
    sig = lambda x: 1.0 / (1.0 + math.exp(-x))
    assert got == pytest.approx([100.0 + 1000.0 * sig(2.0), 40.0 + 4000.0 * sig(4.0), 0.0])


def test_plain_model_reads_one_norm_twice_and_borrows_weights():
    cfg = zc.config("a")
    raw, w = cfg.to_dict(), P.widen(zc.weights(cfg, 1))
    toks = [3, 5, 7, 200]
    logits, layers = P.forward(raw, w, toks, return_layers=True)
    x = layers[2]
    h = P.centred_norm(x, w["l0.norm1"], cfg.eps)
    assert torch.allclose(layers[3], x + P.parallel(cfg.layers[0]["mixer"], w, "l0.mix.", h, cfg.eps)
                          + P.mixture(cfg.layers[0]["mlp"], w, "l0.mlp.", h))
    assert torch.allclose(logits, P.centred_norm(layers[-1], w["final.norm"], cfg.eps) @ w["embed"].T)
    assert not any(k.startswith(("l3.", "l4.")) for k in w)


# ---------------------------------------------------------------- configuration and weights

def test_config_reads_the_nested_keys_and_names_the_one_at_fault(tmp_path):
    cfg = zc.config("a")
    spec = zudusun_spec(cfg)
    assert [l.mixer.kind for l in spec.layers] == ["side_by_side", "attention", "retention"]
    assert [c.layer for c in spec.schedule] == [0, 1, 2, 0, 1] and [l.prefix for l in spec.layers] == ["l0.", "l1.", "l2."]
    b = zudusun_spec(zc.config("b"))
    assert [c.layer for c in b.schedule] == [2, 0, 1, 2, 2] and [l.prefix for l in b.layers] == ["l1.", "l2.", "l4."]
    assert [l.feed_forward.kind for l in b.layers] == ["mixture", "none", "mixture"]
    assert len({cid for _, cid, _ in b.resolved_schedule()}) == 5        # a cache of its own for every layer
    folder = write_random_model(cfg, str(tmp_path / "m"), 0, dtype="float32")
    arch, read = read_config(folder)
    assert arch.name == "Zudusun" and read.layers == cfg.layers and read.to_dict() == dict(cfg.to_dict(), torch_dtype="float32")
    raw = json.load(open(os.path.join(folder, "config.json")))

    def broken(change):
        r = json.loads(json.dumps(raw))
        change(r)
        return r
    for change, text in ((lambda r: r["norm"].pop("eps"), "norm.eps"),
                         (lambda r: r["layers"][2].update(type="other"), r"layers\[2\].type"),
                         (lambda r: r["layers"][0].pop("mixer"), r"layers\[0\].mixer"),
                         (lambda r: r["layers"][0]["mixer"].pop("left"), r"mixer.left.heads"),
                         (lambda r: r["layers"][0]["mixer"]["left"].pop("scale"), r"mixer.left.scale"),
                         (lambda r: r["layers"][0]["mixer"]["right"].pop("tau"), r"mixer.right.tau"),
                         (lambda r: r["layers"][0]["mixer"]["right"].update(tau=-1.0), r"mixer.right.tau"),
                         (lambda r: r["layers"][0]["mixer"].pop("right_scale"), r"mixer.right_scale"),
                         (lambda r: r["layers"][1]["mixer"].update(kv_heads=4), r"layers\[1\].mixer.heads"),
                         (lambda r: r["layers"][1]["mixer"]["mask"].update(size=0), r"mixer.mask.size"),
                         (lambda r: r["layers"][1]["mixer"]["rot"].update(dims=34), r"mixer.rot.dims"),
                         (lambda r: r["layers"][1]["mixer"]["rot"].update(dims=3), r"mixer.rot.dims"),
                         (lambda r: r["layers"][2]["mixer"].update(decay=[0.5]), r"layers\[2\].mixer.decay"),
                         (lambda r: r["layers"][2]["mixer"].update(decay=[0.5, 1.5]), r"layers\[2\].mixer.decay"),
                         (lambda r: r["layers"][2]["mixer"]["rot"].pop("base"), r"mixer.rot.base"),
                         (lambda r: r["layers"][0]["mlp"]["router"].update(top=6), "router.top"),
                         (lambda r: r["layers"][0]["mlp"]["expert"].pop("ff"), "expert.ff"),
                         (lambda r: r["layers"][0]["mlp"]["shared"].pop("ff"), "shared.ff"),
                         (lambda r: r["layers"][0]["mlp"].update(kind="dense"), r"layers\[0\].mlp.kind"),
                         (lambda r: r["layers"][3].update(weights_of=1), r"layers\[3\].weights_of"),
                         (lambda r: r["layers"][3].update(weights_of=9), r"layers\[3\].weights_of"),
                         (lambda r: r["layers"][3].update(weights_of=3), r"weights_of"),
                         (lambda r: r["layers"][0].update(weights_of=3), r"weights_of"),
                         (lambda r: r["layers"][3]["mlp"]["expert"].update(ff=8), r"layers\[3\].weights_of"),
                         (lambda r: r.pop("width"), "width")):
        with pytest.raises(ConfigError, match=text):
            ZudusunConfig.from_dict(broken(change))


def test_the_loader_takes_the_bottleneck_from_the_file_and_names_what_is_missing(tmp_path):
    from safetensors.torch import load_file, save_file
    from transformers_neuronx_amd.engine.factory import runner_from_folder
    cfg = zc.config("a")
    folder = write_random_model(cfg, str(tmp_path / "m"), 0, dtype="float32")
    file = os.path.join(folder, "model.safetensors")
    t = load_file(file)
    shapes = {"embed": (211, 96), "final.norm": (96,), "l0.norm1": (96,), "l0.mix.left.q": (64, 96), "l0.mix.left.v": (48, 96),
              "l0.mix.left.o": (96, 96), "l0.mix.right.q": (36, 96), "l0.mix.right.v": (60, 96), "l0.mix.right.g": (60, 96),
              "l0.mix.right.a1": (5, 96), "l0.mix.right.a2": (36, 5), "l0.mix.right.a2.b": (36,), "l0.mix.right.norm": (20,),
              "l0.mlp.router": (5, 96), "l0.mlp.router.b": (5,), "l0.mlp.e4.up": (24, 96), "l0.mlp.e4.down": (96, 24),
              "l0.mlp.shared.up": (40, 96), "l0.mlp.shared.sg": (1, 96), "l1.mix.q": (192, 96), "l1.mix.q.b": (192,),
              "l1.mix.v.b": (32,), "l1.mix.o.b": (96,), "l1.mix.q.norm": (32,), "l1.mix.k.norm": (32,), "l2.mix.g": (32, 96),
              "l2.mix.o": (96, 32)}
    for name, shape in shapes.items():
        assert tuple(t[name].shape) == shape, name
    assert not any(n.startswith(("l3.", "l4.", "head")) for n in t) and "l0.norm2" not in t
    ecfg = EngineConfig(dtype="float32", kernels="reference", device="cpu", max_tokens=64)
    raw = json.load(open(os.path.join(folder, "config.json")))
    for l in raw["layers"]:
        if l["type"] == "parallel":
            del l["mixer"]["right"]["rank"]           # as a checkpoint's own config.json: the tensor's shape says it
    json.dump(raw, open(os.path.join(folder, "config.json"), "w"))
    toks = [5, 200, 17]
    got = runner_from_folder(folder, ecfg).step([StepEntry("r", toks, [0, 1, 2])])
    want = P.forward(raw, P.widen(t), toks)
    assert float((got.double() - want).abs().max() / want.abs().max()) < TOL
    bad = dict(t)
    del bad["l2.mix.g"]
    bad["l3.norm1"] = torch.zeros(96)
    save_file(bad, file)
    with pytest.raises(WeightsError) as e:
        runner_from_folder(folder, ecfg)
    assert "l2.mix.g" in str(e.value) and "l3.norm1" in str(e.value)
    save_file(dict(t, **{"l0.mix.right.a2": torch.zeros(36, 4)}), file)
    with pytest.raises(ValueError, match="a2"):
        runner_from_folder(folder, ecfg)


def test_parts_refuse_what_they_cannot_be():
    from transformers_neuronx_amd.parts.base import FEED_FORWARDS, MIXERS
    from transformers_neuronx_amd.parts.spec import PartSpec
    moe = dict(width=8, experts=2, top=1, inner=4, router_name="router", expert_name="e{}.", gated=False, activation="relu2",
               names=("up", "down"))
    FEED_FORWARDS.build(PartSpec("mixture", moe))
    for change in (dict(weight_on="input"), dict(names=("gate", "up", "down")), dict(activation="silu"),
                   dict(gated=True, activation="silu", names=("gate", "up", "down"), shared_inner=4, shared_gate_name="sg")):
        with pytest.raises(ValueError):
            FEED_FORWARDS.build(PartSpec("mixture", dict(moe, **change)))
    ret = dict(width=8, heads=2, head_size=4, value_size=4, decay=(0.5, 0.9), eps=1e-5, names=("q", "k", "v", "g", "o"))
    MIXERS.build(PartSpec("retention", ret))
    for change in (dict(decay=(0.5,)), dict(decay=(0.5, 0.0)), dict(head_size=300), dict(names=("q", "k", "v", "o"))):
        with pytest.raises(ValueError):
            MIXERS.build(PartSpec("retention", dict(ret, **change)))
    with pytest.raises(ValueError, match="tensor or a number"):
        MIXERS.build(PartSpec("attention", dict(width=8, num_heads=1, head_size=16, names=("q", "k", "v", "o"), sink="s", sink_score=0.0)))


# ---------------------------------------------------------------- the engine on the host

def _expected(cfg, w, requests):
    raw, wide = cfg.to_dict(), P.widen(w)
    return {rid: P.forward(raw, wide, toks) for rid, toks in requests.items()}


def step_through(runner, expected, made, tol, few_over=0.0):
    """`few_over`: the share of positions that may lie over `tol`, by any distance: in bfloat16 a rounding of the
    router's input changes which expert a token takes where two logits are close, and that token's result is another
    expert's. float32 allows none."""
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


@pytest.mark.parametrize("name", ["a", "b"])
def test_the_stream_after_every_layer(name):
    from transformers_neuronx_amd import debug
    cfg = zc.config(name)
    w = zc.weights(cfg, 2)
    toks = zc.requests(cfg, [19], 0)["r0"]
    _, layers = P.forward(cfg.to_dict(), P.widen(w), toks, return_layers=True)
    runner = zc.runner(cfg, w)
    with debug.debug_context() as taps:
        runner.step([StepEntry("r0", toks, [])])
    for i, want in enumerate(layers):
        got = taps[f"call{i}.layer{runner.model.schedule[i][0]}"]
        assert float((got.double() - want).abs().max() / want.abs().max()) < 1e-5, i


@pytest.mark.parametrize("name", sorted(zc.CASES))
def test_schedules_on_the_host(name):
    cfg = zc.config(name)
    w = zc.weights(cfg, 3)
    runner = zc.runner(cfg, w, max_tokens=208)
    requests = zc.requests(cfg, [70, 33, 5, 100, 1], 1)
    expected = _expected(cfg, w, requests)
    for made in (schedules.whole(requests), schedules.head_then_singles(requests, tail=12), schedules.portions(requests),
                 schedules.portions(requests, sizes=(2, 2, 3, 2, 16, 2, 15, 17, 2)),
                 schedules.mixed(requests, max_tokens=208, page=16, seed=5, tail=8, max_live=3),
                 schedules.only_last(schedules.mixed(requests, max_tokens=208, page=16, seed=6, tail=20, max_live=4))):
        step_through(runner, expected, made, TOL)


def test_pages_and_slots_that_are_used_again():
    """One request at a time in a pool that holds one: every request gets the pages and the slot the one before left
    full."""
    cfg = zc.config("b")
    w = zc.weights(cfg, 4)
    runner = zc.runner(cfg, w, max_tokens=48, max_seqs=1)
    requests = zc.requests(cfg, [37, 20, 3, 45], 2)
    expected = _expected(cfg, w, requests)
    for rid, toks in requests.items():
        assert all(g.pool.num_free == g.pool.num_pages for g in runner.cache.groups.values())
        got = runner.step([StepEntry(rid, toks[:2], [0, 1])])
        got = torch.cat([got, runner.step([StepEntry(rid, toks[2:], list(range(len(toks) - 2)))])])
        assert float((got.double() - expected[rid]).abs().max() / expected[rid].abs().max()) < TOL
        runner.finish(rid)


@pytest.mark.parametrize("name", ["a", "b"])
def test_one_product_for_all_that_reads_a_norm_is_the_products_of_each(name):
    """The same model with the parts' input products apart, and the joined matrix's rows as the parts laid them."""
    from dataclasses import replace
    from transformers_neuronx_amd.engine.model import DecoderModel
    from transformers_neuronx_amd.kernels import make_ops
    from transformers_neuronx_amd.parts.spec import PartSpec
    from transformers_neuronx_amd.weights.loader import TensorDict
    cfg = zc.config(name)
    w = zc.weights(cfg, 7)
    runner = zc.runner(cfg, w)
    toks = zc.requests(cfg, [25], 0)["r0"]
    got = runner.step([StepEntry("r", toks, list(range(25)))])
    spec = zudusun_spec(cfg)
    apart = DecoderModel(replace(spec, layers=tuple(replace(l, block=PartSpec("parallel", {})) for l in spec.layers)))
    ops = make_ops("reference", torch.float32, "cpu")
    apart.load(TensorDict({k: v.clone() for k, v in w.items()}), ops, torch.float32, torch.device("cpu"))
    assert any(l.block.joins for l in runner.model.layers) and not any(l.block.joins for l in apart.layers)
    for layer in runner.model.layers:
        if layer.block.joins:
            matrix = layer.block.w_in
            assert matrix.shape[0] % 16 == 0 and all(a % 16 == 0 for a, _ in layer.block.places)
            assert not hasattr(layer.mixer, "w_in") and not hasattr(layer.feed_forward, "w_in")
        else:
            assert layer.mixer.w_in is not None
    runner.finish("r")
    runner.model = apart
    other = runner.step([StepEntry("r", toks, list(range(25)))])
    assert float((got - other).abs().max() / got.abs().max()) < 1e-5


def test_rows_a_power_of_two_apart_are_moved():
    from types import SimpleNamespace
    from transformers_neuronx_amd.parts.base import joined_rows
    part = lambda rows, bias: SimpleNamespace(in_matrix=lambda: (torch.full((rows, 3), float(rows)), bias))
    w, bias, places = joined_rows((part(5, None), part(1000, torch.ones(1000))))
    assert places == [(0, 5), (16, 1016)] and w.shape == (1024 + 64, 3)
    assert float(w[:5].mean()) == 5.0 and float(w[16:1016].mean()) == 1000.0 and float(w[5:16].abs().sum() + w[1016:].abs().sum()) == 0
    assert float(bias[16:1016].sum()) == 1000.0 and float(bias.sum()) == 1000.0
    w, bias, _ = joined_rows((part(5, None), part(7, None)))
    assert bias is None and w.shape == (32, 3)


def test_layers_with_the_same_weights_keep_caches_of_their_own():
    cfg = zc.config("b")
    runner = zc.runner(cfg, zc.weights(cfg, 4))
    calls = runner.model.schedule
    assert len({cid for _, cid, _ in calls}) == len(calls)
    runner.step([StepEntry("r", [1, 2, 3], [])])
    slot_of = [runner.cache.caches[calls[i][1]].state["memory"] for i in (0, 3, 4)]
    assert all(float(s.abs().max()) > 0 for s in slot_of)
    assert not torch.equal(slot_of[0], slot_of[1]) and not torch.equal(slot_of[1], slot_of[2])


def test_long_decoding_on_the_host():
    cfg = zc.config("d")
    w = zc.weights(cfg, 5)
    runner = zc.runner(cfg, w, max_tokens=160, max_seqs=2)
    toks = zc.requests(cfg, [150], 3)["r0"]
    expected = _expected(cfg, w, {"r0": toks})["r0"]
    got = [runner.step([StepEntry("r0", toks[:3], list(range(3)))])]
    for t in toks[3:]:
        got.append(runner.step([StepEntry("r0", [t], [0])]))
    got = torch.cat(got)
    assert float((got.double() - expected).abs().max() / expected.abs().max()) < TOL


def _greedy(cfg, w, prompt, new):
    raw, wide = cfg.to_dict(), P.widen(w)
    toks = list(prompt)
    for _ in range(new):
        toks.append(int(P.forward(raw, wide, toks)[-1].argmax()))
    return toks[len(prompt):]


@pytest.mark.parametrize("run_ahead", [False, True])
def test_greedy_generation_through_the_scheduler(run_ahead):
    cfg = zc.config("b")
    w = zc.weights(cfg, 6)
    ecfg = EngineConfig(dtype="float32", kernels="reference", device="cpu", page_size=16, max_tokens=96, max_num_seqs=3,
                        max_num_batched_tokens=24, chunk_size=9, run_ahead=run_ahead)
    from transformers_neuronx_amd.engine.factory import build_runner
    from transformers_neuronx_amd.weights.loader import TensorDict
    engine = LLMEngine(build_runner(cfg, TensorDict(w), ecfg), ecfg)
    prompts = list(zc.requests(cfg, [30, 3, 17, 1, 22], 7).values())
    out = engine.generate(prompts, SamplingParams(temperature=0.0, max_new_tokens=12, ignore_eos=True))
    for prompt, tokens in zip(prompts, out):
        assert tokens == _greedy(cfg, w, prompt, 12)
    engine.runner.cache.check()
    assert not engine.runner.cache.requests


def test_generation_through_the_entry_point_on_the_host(tmp_path):
    from safetensors.torch import load_file
    from transformers_neuronx_amd import NeuronAutoModelForCausalLM
    from transformers_neuronx_amd.zudusun.model import ZudusunForSampling
    cfg = zc.config("a")
    folder = write_random_model(cfg, str(tmp_path / "m"), 11, dtype="float32")
    w = load_file(os.path.join(folder, "model.safetensors"))
    model = NeuronAutoModelForCausalLM.from_pretrained(folder, batch_size=2, amp="f32", n_positions=64, page_size=16,
                                                       kernels="reference", device="cpu")
    assert type(model) is ZudusunForSampling
    model.to_neuron()
    ids = torch.tensor([[5, 200, 17, 3], [9, 9, 100, 42]])
    out = model.sample(ids, sequence_length=14, top_k=1)
    for row in range(2):
        assert out[row, 4:].tolist() == _greedy(cfg, w, ids[row].tolist(), 10)


@pytest.mark.parametrize("seed", range(10))
def test_configurations_drawn_from_a_seed_on_the_host(seed):
    cfg = zc.drawn(seed)
    w = zc.weights(cfg, seed)
    runner = zc.runner(cfg, w, max_tokens=176)
    requests = zc.requests(cfg, [70, 33, 5, 1], seed)
    step_through(runner, _expected(cfg, w, requests), schedules.mixed(requests, max_tokens=176, page=16, seed=5, tail=8, max_live=3), TOL)
