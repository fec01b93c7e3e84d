"""Small Gubulorn configurations of the tests' own, their random weights, and the runner that serves them. The sizes
differ between the cases in everything that can differ: either kind of layer first and last, grouped and ungrouped
heads in both mixers, value heads smaller and larger than query heads, state spaces of 3 elements and more, one and
several norm groups, convolutions of 1 to 5 taps, temperatures that grow at every token, at every few, and not at all,
dense, routed and no feed-forwards, with and without experts that have no tensors, one group and several, one expert a
token and several, with and without a cap on the logits, widths that are multiples of nothing."""
import random

import torch

from transformers_neuronx_amd.config import EngineConfig
from transformers_neuronx_amd.engine.factory import build_runner
from transformers_neuronx_amd.engine.model import model_param_decls
from transformers_neuronx_amd.gubulorn import GubulornConfig, gubulorn_spec
from transformers_neuronx_amd.weights.loader import TensorDict
from transformers_neuronx_amd.weights.random_init import random_tensors


def delta(heads, kv_heads, dim, vdim, conv):
    return "delta", dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, conv=conv)


def parallel(left, right):
    """left = (heads, kv_heads, dim, vdim, scale, temperature or None), right = (heads, vdim, state, groups, conv,
    norm_groups)."""
    heads, kv_heads, dim, vdim, scale, temp = left
    a = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale)
    if temp is not None:
        a["q_temp"] = dict(coef=temp[0], every=temp[1])
    keys = ("heads", "vdim", "state", "groups", "conv", "norm_groups")
    return "parallel", dict(left=a, right=dict(zip(keys, right)))


def dense(ff, limit):
    return dict(kind="dense", ff=ff, limit=limit)


def moe(experts, identity, top, ff, count=1, keep=1):
    return dict(kind="moe", router=dict(experts=experts, identity=identity, top=top, groups=dict(count=count, keep=keep)),
                expert=dict(ff=ff))


def layer(mixer, mlp):
    return dict(type=mixer[0], mixer=mixer[1], mlp=mlp)


CASES = {
    # the delta rule first, the pair last; a layer without a feed-forward
    "a": dict(architecture="Gubulorn", vocab=211, width=96, norm=dict(eps=1e-4), postln_alpha=2.6, logit_scale=0.75,
              logit_softcap=9.0,
              layers=[layer(delta(4, 2, 16, 24, 4), moe(5, 3, 3, 40, 4, 2)),
                      layer(parallel((6, 2, 16, 32, 0.3, (0.4, 7)), (4, 8, 24, 2, 3, 1)), dense(72, 0.8)),
                      layer(delta(3, 3, 24, 8, 2), None),
                      layer(parallel((4, 4, 32, 16, 0.2, (0.7, 1)), (6, 16, 8, 3, 4, 4)), moe(6, 2, 1, 24, 2, 1))]),
    # the pair first; sizes that are multiples of nothing; a convolution of one tap (no inputs kept) and of five
    "b": dict(architecture="Gubulorn", vocab=77, width=50, norm=dict(eps=1e-4), postln_alpha=3.2,
              layers=[layer(parallel((3, 1, 10, 6, 0.25, None), (5, 7, 3, 1, 5, 5)), moe(7, 0, 4, 26)),
                      layer(delta(2, 1, 10, 14, 1), dense(30, 2.0)),
                      layer(parallel((2, 2, 20, 21, 0.4, (0.2, 3)), (3, 10, 18, 3, 1, 2)), moe(3, 4, 2, 16, 7, 3)),
                      layer(delta(6, 3, 5, 3, 3), moe(4, 4, 2, 10, 2, 1))]),
    # sizes the matrix-unit kernels take: multiples of 16, a 64 and a 128 among the heads
    "c": dict(architecture="Gubulorn", vocab=320, width=128, norm=dict(eps=1e-5), postln_alpha=3.0, logit_scale=1.0,
              logit_softcap=20.0,
              layers=[layer(parallel((4, 2, 64, 64, 0.12, (0.3, 20)), (8, 16, 64, 2, 4, 2)), dense(256, 1.5)),
                      layer(delta(2, 2, 128, 64, 4), moe(6, 2, 2, 64, 4, 2)),
                      layer(delta(8, 4, 64, 32, 3), dense(128, 1.0)),
                      layer(parallel((8, 1, 32, 16, 0.2, (0.5, 5)), (4, 64, 128, 1, 2, 8)), moe(12, 4, 4, 32, 4, 2))]),
    # one layer of each kind, values the other cases make unequal or other than 1
    "d": dict(architecture="Gubulorn", vocab=130, width=64, norm=dict(eps=1e-3), postln_alpha=1.0, logit_scale=1.0,
              layers=[layer(parallel((1, 1, 16, 16, 1.0, (1.0, 1)), (1, 16, 16, 1, 1, 1)), moe(1, 1, 1, 48, 1, 1)),
                      layer(delta(1, 1, 16, 16, 1), dense(8, 1.0))]),
}


def config(name) -> GubulornConfig:
    return GubulornConfig.from_dict(dict(CASES[name], init_std=0.35))


def weights(cfg, seed, storage=torch.float32):
    """Random tensors by checkpoint name (matrices in `storage`), made lively: wide enough that no part drowns, memories
    that remember a few tokens and some that remember hundreds, sinks that weigh about as much as a key, corrections
    that change which experts are chosen (some large enough that choice scores are negative), clamps that are met."""
    w = random_tensors(model_param_decls(gubulorn_spec(cfg)), cfg.init_std, seed, storage)
    g = torch.Generator().manual_seed(seed + 1000)
    for k in list(w):
        last = k.rsplit(".", 1)[-1]
        if last == "conv" or k.endswith("conv.b"):
            w[k] = torch.randn(w[k].shape, generator=g) * 0.7
        elif w[k].dim() == 2 and last in ("q", "k", "v", "o", "in", "gate", "up", "down", "head"):
            w[k] = (w[k].float() * (1.5 / w[k].shape[1] ** 0.5 / cfg.init_std)).to(w[k].dtype)
        elif w[k].dim() == 2 and last in ("g", "a", "b", "router"):
            w[k] = (w[k].float() * (2.5 / w[k].shape[1] ** 0.5 / cfg.init_std)).to(w[k].dtype)
        elif last == "A_log":
            w[k] = torch.randn(w[k].shape, generator=g) * 1.5 - 1.0
        elif last == "dt_bias":
            w[k] = torch.randn(w[k].shape, generator=g) * 1.5 - 1.0
        elif last == "sink":
            w[k] = torch.randn(w[k].shape, generator=g) * 1.5
        elif last == "correction":
            w[k] = torch.randn(w[k].shape, generator=g) * 0.25
    return w


def runner(cfg, w, dtype="float32", kernels="reference", device="cpu", page_size=16, max_tokens=256, max_seqs=4,
           use_graphs=True):
    ecfg = EngineConfig(dtype=dtype, page_size=page_size, max_tokens=max_tokens, max_num_seqs=max_seqs, device=device,
                        kernels=kernels, use_graphs=use_graphs)
    return build_runner(cfg, TensorDict({k: v.clone() for k, v in w.items()}), ecfg)


def requests(cfg, lengths, seed):
    g = torch.Generator().manual_seed(seed)
    return {f"r{i}": torch.randint(0, cfg.vocab, (n,), generator=g).tolist() for i, n in enumerate(lengths)}


def drawn(seed: int) -> GubulornConfig:
    """A configuration drawn from a seed: any sizes, any order of the two kinds of layers, any feed-forward or none."""
    rnd = random.Random(seed)
    width = rnd.choice([24, 36, 64, 100, 128, 256])
    layers = []
    for i in range(rnd.randint(1, 5)):
        if rnd.random() < 0.5:
            groups = rnd.choice([1, 2, 3])
            mixer = delta(groups * rnd.choice([1, 2, 4]), groups, rnd.choice([4, 10, 16, 32, 64, 96, 128]),
                          rnd.choice([3, 8, 16, 24, 64]), rnd.choice([1, 2, 3, 4, 5, 7]))
        else:
            kv, groups = rnd.choice([1, 2, 3]), rnd.choice([1, 2, 3])
            heads, vdim = groups * rnd.choice([1, 2, 4]), rnd.choice([4, 6, 16, 32, 64])
            parts = rnd.choice([p for p in range(1, heads * vdim + 1) if heads * vdim % p == 0 and heads * vdim // p >= 8 or p == 1])
            mixer = parallel((kv * rnd.choice([1, 2, 4, 6]), kv, rnd.choice([4, 10, 16, 32, 64, 96]),
                              rnd.choice([4, 10, 16, 48, 64]), rnd.uniform(0.05, 0.4),
                              rnd.choice([None, (0.5, 1), (0.3, 4), (0.2, 50)])),
                             (heads, vdim, rnd.choice([3, 8, 16, 40, 64, 128]), groups, rnd.choice([1, 2, 3, 4, 6]), parts))
        kind = rnd.random()
        if kind < 0.15:
            mlp = None
        elif kind < 0.45:
            mlp = dense(rnd.choice([8, 20, 64, 200]), rnd.choice([0.5, 1.0, 7.0]))
        else:
            count = rnd.choice([1, 1, 2, 3, 5])
            per = rnd.choice([1, 2, 4, 14])
            keep = rnd.randint(1, count)
            identity = rnd.randint(0, (count * per) // 2)
            mlp = moe(count * per - identity, identity, rnd.randint(1, min(keep * per, 5)), rnd.choice([8, 20, 64, 72]), count, keep)
        layers.append(layer(mixer, mlp))
    raw = dict(architecture="Gubulorn", vocab=rnd.choice([50, 97, 256, 300]), width=width,
               norm=dict(eps=rnd.choice([1e-5, 1e-4, 1e-3])), postln_alpha=rnd.choice([2.4, 2.7, 3.0, 3.3]), layers=layers,
               init_std=0.35)
    if rnd.random() < 0.7:
        raw["logit_scale"] = rnd.choice([0.25, 1.0, 2.0])
    if rnd.random() < 0.7:
        raw["logit_softcap"] = rnd.choice([2.0, 10.0, 40.0])
    return GubulornConfig.from_dict(raw)
