"""Small Zudusun configurations of the tests' own, their random weights, and the runner that serves them. The sizes
differ between the cases in everything that can differ: each kind of layer first and last, layers that run with the
weights of an earlier layer, of a later one and of one that itself borrows, grouped and ungrouped heads, value heads
smaller and larger than query heads and equal to them, heads wholly and partly turned and not at all, windows of one
token up to more than a request, decays near 0 and 1, bottlenecks of one element and of many, one expert a token and
all of them, with and without a shared expert, layers without a feed-forward, widths that are multiples of nothing."""
import random

import torch

from transformers_neuronx_amd.config import EngineConfig
from transformers_neuronx_amd.engine.factory import build_runner
from transformers_neuronx_amd.engine.model import model_param_decls
from transformers_neuronx_amd.weights.loader import TensorDict
from transformers_neuronx_amd.weights.random_init import random_tensors
from transformers_neuronx_amd.zudusun import ZudusunConfig, zudusun_spec


def parallel(left, right, scales=(0.7, 0.6)):
    """left = (heads, kv_heads, dim, vdim, scale), right = (heads, dim, vdim, tau, rank)."""
    return "parallel", dict(left=dict(zip(("heads", "kv_heads", "dim", "vdim", "scale"), left)),
                            right=dict(zip(("heads", "dim", "vdim", "tau", "rank"), right)),
                            left_scale=scales[0], right_scale=scales[1])


def attention(heads, kv_heads, dim, vdim, scale, window, base, dims):
    return "attention", dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale, mask=dict(size=window),
                             rot=dict(base=base, dims=dims))


def retention(heads, dim, vdim, decay, base, dims):
    return "retention", dict(heads=heads, dim=dim, vdim=vdim, decay=list(decay), rot=dict(base=base, dims=dims))


def moe(experts, top, ff, shared=None):
    m = dict(kind="moe", router=dict(experts=experts, top=top), expert=dict(ff=ff))
    if shared is not None:
        m["shared"] = dict(ff=shared)
    return m


def layer(mixer, mlp, weights_of=None):
    d = dict(type=mixer[0], mixer=mixer[1], mlp=mlp)
    if weights_of is not None:
        d["weights_of"] = weights_of
    return d


_A0 = (parallel((4, 2, 16, 24, 0.3), (3, 12, 20, 8.0, 5)), moe(5, 2, 24, 40))
_A1 = (attention(6, 2, 32, 16, 0.25, 20, 500.0, 12), moe(7, 3, 16, 8))
_B0 = (retention(3, 10, 7, (0.9, 0.99, 0.5), 100.0, 4), moe(3, 3, 26, 30))
_B2 = (parallel((3, 1, 10, 6, -0.4), (5, 7, 3, 1.0, 1), (1.0, -0.5)), None)
_C1 = (parallel((4, 1, 128, 128, 0.1), (2, 128, 64, 16.0, 16), (0.5, 1.0)), moe(6, 2, 64, 128))

CASES = {
    # each kind once, then the first two again with their weights
    "a": dict(architecture="Zudusun", vocab=211, width=96, norm=dict(eps=1e-4),
              layers=[layer(*_A0), layer(*_A1), layer(retention(2, 24, 16, (0.97, 0.9995), 1e4, 24), moe(4, 1, 40, 16)),
                      layer(*_A0, weights_of=0), layer(*_A1, weights_of=1)]),
    # sizes that are multiples of nothing; the weights of a layer that comes later, and of one that borrows them itself;
    # a layer without a feed-forward, one without a shared expert; a window of one token
    "b": dict(architecture="Zudusun", vocab=77, width=50, norm=dict(eps=1e-3),
              layers=[layer(*_B0, weights_of=4), layer(attention(3, 3, 10, 14, 0.5, 1, 30.0, 10), moe(4, 2, 10)),
                      layer(*_B2), layer(*_B0, weights_of=0), layer(*_B0)]),
    # sizes the matrix-unit kernels take: multiples of 16, a 64 and a 128 among the heads
    "c": dict(architecture="Zudusun", vocab=320, width=128, norm=dict(eps=1e-5),
              layers=[layer(attention(4, 2, 64, 64, 0.12, 100, 1e4, 64), moe(8, 4, 64, 96)), layer(*_C1),
                      layer(retention(2, 64, 128, (0.998, 0.9), 1e5, 32), moe(6, 6, 32, 64)), layer(*_C1, weights_of=1),
                      layer(attention(8, 1, 32, 48, 0.2, 33, 1e3, 16), moe(12, 1, 64, 64))]),
    # values the other cases make unequal or other than 1
    "d": dict(architecture="Zudusun", vocab=130, width=64, norm=dict(eps=1e-5),
              layers=[layer(retention(1, 16, 16, (1.0,), 1e4, 0), moe(1, 1, 48, 48)),
                      layer(parallel((1, 1, 16, 16, 1.0), (1, 16, 16, 1.0, 16), (1.0, 1.0)), moe(1, 1, 8)),
                      layer(attention(1, 1, 16, 16, 1.0, 500, 1e4, 0), None)]),
}


def config(name) -> ZudusunConfig:
    return ZudusunConfig.from_dict(dict(CASES[name], init_std=0.35))


def weights(cfg, seed, storage=torch.float32):
    """Random tensors by checkpoint name (matrices in `storage`), made lively: wide enough that no part drowns, key
    channels that remember a few tokens and some that remember hundreds, biases of the router that change the choice."""
    w = random_tensors(model_param_decls(zudusun_spec(cfg)), cfg.init_std, seed, storage)
    g = torch.Generator().manual_seed(seed + 1000)
    for k in list(w):
        last = k.rsplit(".", 1)[-1]
        if k == "embed":
            w[k] = torch.randn(w[k].shape, generator=g).to(w[k].dtype)
        elif w[k].dim() == 2 and last in ("q", "k", "v", "o", "up", "down"):
            w[k] = (w[k].float() * (1.5 / w[k].shape[1] ** 0.5 / cfg.init_std)).to(w[k].dtype)
        elif w[k].dim() == 2 and last in ("g", "a1", "a2", "router", "sg"):
            w[k] = (w[k].float() * (2.5 / w[k].shape[1] ** 0.5 / cfg.init_std)).to(w[k].dtype)
        elif k.endswith("a2.b"):
            w[k] = torch.randn(w[k].shape, generator=g) * 2.0 + 2.0
    return w


def runner(cfg, w, dtype="float32", kernels="reference", device="cpu", page_size=16, max_tokens=256, max_seqs=4,
           use_graphs=True):
    ecfg = EngineConfig(dtype=dtype, page_size=page_size, max_tokens=max_tokens, max_num_seqs=max_seqs, device=device,
                        kernels=kernels, use_graphs=use_graphs)
    return build_runner(cfg, TensorDict({k: v.clone() for k, v in w.items()}), ecfg)


def requests(cfg, lengths, seed):
    g = torch.Generator().manual_seed(seed)
    return {f"r{i}": torch.randint(0, cfg.vocab, (n,), generator=g).tolist() for i, n in enumerate(lengths)}


def drawn(seed: int) -> ZudusunConfig:
    """A configuration drawn from a seed: any sizes, any order of the three kinds of layers, borrowed weights, any
    feed-forward or none."""
    rnd = random.Random(seed)
    width = rnd.choice([24, 36, 64, 100, 128, 256])
    layers = []
    for i in range(rnd.randint(1, 6)):
        if layers and rnd.random() < 0.25:
            j = rnd.randrange(len(layers))
            layers.append(dict(layers[j], weights_of=j))
            continue
        kind = rnd.random()
        if kind < 0.4:
            kv = rnd.choice([1, 2, 3])
            mixer = parallel((kv * rnd.choice([1, 2, 4]), kv, rnd.choice([4, 10, 16, 32, 64, 96]), rnd.choice([4, 16, 48, 64]),
                              rnd.uniform(0.05, 0.4)),
                             (rnd.choice([1, 2, 3, 4]), rnd.choice([3, 8, 16, 40, 64, 128]), rnd.choice([4, 10, 16, 64]),
                              rnd.choice([0.5, 1.0, 4.0, 16.0]), rnd.choice([1, 3, 8, 16, 20])),
                             (rnd.uniform(0.3, 1.0), rnd.uniform(0.3, 1.0)))
        elif kind < 0.7:
            kv, dim = rnd.choice([1, 2, 3]), rnd.choice([4, 10, 16, 32, 64, 128])
            mixer = attention(kv * rnd.choice([1, 2, 4, 6]), kv, dim, rnd.choice([4, 10, 16, 48, 64, 128]), rnd.uniform(0.05, 0.4),
                              rnd.choice([1, 2, 15, 16, 17, 40, 300]), rnd.choice([10.0, 1e3, 1e4]), 2 * rnd.randint(0, dim // 2))
        else:
            heads, dim = rnd.choice([1, 2, 5]), rnd.choice([4, 10, 16, 32, 64, 128])
            mixer = retention(heads, dim, rnd.choice([3, 16, 24, 64]), [1.0 - 10 ** rnd.uniform(-4, -0.3) for _ in range(heads)],
                              rnd.choice([10.0, 1e3, 1e4]), 2 * rnd.randint(0, dim // 2))
        experts = rnd.choice([1, 2, 3, 8, 20])
        mlp = None if rnd.random() < 0.15 else moe(experts, rnd.randint(1, min(experts, 5)), rnd.choice([8, 20, 64, 72]),
                                                   rnd.choice([None, 8, 20, 64]))
        layers.append(layer(mixer, mlp))
    return ZudusunConfig.from_dict(dict(architecture="Zudusun", vocab=rnd.choice([50, 97, 256, 300]), width=width,
                                        norm=dict(eps=rnd.choice([1e-5, 1e-4, 1e-3])), layers=layers, init_std=0.35))
