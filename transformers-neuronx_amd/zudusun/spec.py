"""Zudusun as a `ModelSpec`: which parts, with which sizes, under which tensor names.

Tensor names: `embed` (the token table and the head), `final.norm`; layer i's start with `l<i>.`: the norm `norm1`, the
mixer's `mix.*` (the two side by side: `left.{q, k, v, o}`, `right.{q, k, v, g, o, a1, a2, a2.b, norm}`; attention: `q`, `k`, `v`,
`o`, each with a bias `.b`, `q.norm`, `k.norm`; retention: `q`, `k`, `v`, `g`, `o`), the feed-forward's `mlp.*` (`router`,
`router.b`, `e<j>.{up, down}`, `shared.{up, down, sg}`). Matrix names carry no suffix. A layer with `weights_of` is a second
call of that layer in the run order, with a cache of its own.
"""
from .config import ZudusunConfig
from ..config.registry import register_architecture
from ..parts.spec import LayerCall, LayerSpec, ModelSpec, PartSpec


def _rotary(m: dict, interleaved: bool):
    rot = m.get("rot")
    if rot is None:
        return None
    return PartSpec("rotary", dict(base=rot["base"], dims=m["dim"] if rot.get("dims") is None else rot["dims"],
                                   interleaved=interleaved))


def _mixer(cfg: ZudusunConfig, kind: str, m: dict) -> PartSpec:
    d, eps = cfg.width, cfg.eps

    def attention(a, **more):
        return PartSpec("attention", dict(
            width=d, num_heads=a["heads"], num_kv_heads=a["heads"] if a.get("kv_heads") is None else a["kv_heads"],
            head_size=a["dim"], value_size=a["vdim"], names=("q", "k", "v", "o"), weight_suffix="", bias_suffix=".b",
            scale=a["scale"], float32_route=True, **more))
    if kind == "parallel":
        r = m["right"]
        right = PartSpec("gated_linear_attention", dict(
            width=d, heads=r["heads"], head_size=r["dim"], value_size=r["vdim"], tau=r["tau"], eps=eps, rank=r.get("rank"),
            names=("q", "k", "v", "g", "o", "a1", "a2", "norm")))
        return PartSpec("side_by_side", dict(left=attention(m["left"], bias=False), right=right, left_scale=m["left_scale"],
                                             right_scale=m["right_scale"]))
    if kind == "attention":
        return attention(m, bias=True, window=(m.get("mask") or {}).get("size"), rotation=_rotary(m, True),
                         qk_norm=dict(eps=eps, suffix=".norm", shared=True), sink_score=0.0)
    return PartSpec("retention", dict(
        width=d, heads=m["heads"], head_size=m["dim"], value_size=m["vdim"], decay=m["decay"], eps=eps,
        names=("q", "k", "v", "g", "o"), rotation=_rotary(m, False)))


def _feed_forward(cfg: ZudusunConfig, mlp) -> PartSpec:
    if mlp is None:
        return PartSpec("none", {})
    shared = mlp.get("shared")
    return PartSpec("mixture", dict(
        width=cfg.width, experts=mlp["router"]["experts"], top=mlp["router"]["top"], inner=mlp["expert"]["ff"],
        shared_inner=shared["ff"] if shared else 0, score="softmax", renormalize=True, weight_on="output",
        activation="relu2", gated=False, router_name="router", router_bias_name="router.b", expert_name="e{}.",
        shared_name="shared.", shared_gate_name="sg", names=("up", "down")))


def zudusun_spec(cfg: ZudusunConfig) -> ModelSpec:
    d = cfg.width
    norm = PartSpec("layer_norm", dict(width=d, eps=cfg.eps, affine=True, bias=False, weight_suffix=""))
    no_norm = PartSpec("layer_norm", dict(width=d, eps=cfg.eps, affine=False))       # a layer has one norm
    layers, place = [], {}
    for i, layer in enumerate(cfg.layers):
        if cfg.owner(i) != i:
            continue
        place[i] = len(layers)
        layers.append(LayerSpec(prefix=f"l{i}.", block=PartSpec("parallel", dict(one_product=True)),
                                mixer=_mixer(cfg, layer["type"], layer["mixer"]),
                                feed_forward=_feed_forward(cfg, layer.get("mlp")), mixer_norm=norm,
                                feed_forward_norm=no_norm, mixer_name="mix.", feed_forward_name="mlp.",
                                mixer_norm_name="norm1", feed_forward_norm_name="norm2"))
    schedule = tuple(LayerCall(place[cfg.owner(i)]) for i in range(len(cfg.layers)))
    embedding = PartSpec("token_table", dict(vocab=cfg.vocab, embed_width=d, width=d, position=PartSpec("none", {}),
                                             table_name="embed", projection_name=None, position_name=None))
    head = PartSpec("vocab_projection", dict(vocab=cfg.vocab, embed_width=d, width=d, norm=norm, weight_name="embed",
                                             tied_to=None, projection_name=None, norm_name="final.norm"))
    return ModelSpec(hidden_size=d, vocab_size=cfg.vocab, max_positions=cfg.max_positions, embedding=embedding,
                     layers=tuple(layers), schedule=schedule, head=head, init_std=cfg.init_std)


ARCHITECTURE = register_architecture("Zudusun", "zudusun", ZudusunConfig, zudusun_spec,
                                     model_class="transformers_neuronx_amd.zudusun.model:ZudusunForSampling")
