"""Gubulorn as a `ModelSpec`: which parts, with which sizes, under which tensor names.

Tensor names: `embed`, `embed.norm`, `final.norm`, `head`; layer i's start with `l<i>.`: the norms `norm1` and `norm2`,
the mixer's `mix.*` (the delta rule: `q`, `k`, `v`, each with `.conv`, `b`, `a`, `g`, `o`, `A_log`, `dt_bias`, `norm`; the two
mixers side by side: `left.{q, k, v, q.norm, k.norm, sink, g, o}`, `right.{in, conv, conv.b, dt_bias, A_log, D, norm, o}`,
`left.out`, `right.out`), the feed-forward's `mlp.*` (dense: `gate`, `up`, `down`; experts: `router`, `correction`,
`e<j>.{gate, up, down}`). Matrix names carry no suffix.
"""
from .config import GubulornConfig
from ..config.registry import register_architecture
from ..parts.spec import LayerSpec, ModelSpec, PartSpec


def _mixer(cfg: GubulornConfig, kind: str, m: dict) -> PartSpec:
    d, eps = cfg.width, cfg.eps
    if kind == "delta":
        return PartSpec("gated_delta", dict(
            width=d, heads=m["heads"], groups=m.get("kv_heads", m["heads"]), head_size=m["dim"], value_size=m["vdim"],
            taps=m["conv"], eps=eps, names=("q", "k", "v", "g", "a", "b", "o", "A_log", "dt_bias", "norm")))
    a, s = m["left"], m["right"]
    left = PartSpec("attention", dict(
        width=d, num_heads=a["heads"], num_kv_heads=a.get("kv_heads", a["heads"]), head_size=a["dim"], value_size=a["vdim"],
        names=("q", "k", "v", "o"), weight_suffix="", bias=False, scale=a["scale"],
        qk_norm=dict(eps=eps, suffix=".norm", shared=True), temperature=a.get("q_temp"), sink="sink", out_gate="g",
        out_gate_per_head=True))
    right = PartSpec("state_space", dict(
        width=d, heads=s["heads"], groups=s["groups"], head_size=s["state"], value_size=s["vdim"], taps=s["conv"],
        norm_groups=s["norm_groups"], eps=eps, names=("in", "conv", "dt_bias", "A_log", "D", "norm", "o")))
    return PartSpec("side_by_side", dict(left=left, right=right, left_scale=0.5, right_scale=0.5,
                                         out_norms=dict(eps=eps, left="left.out", right="right.out")))


def _feed_forward(cfg: GubulornConfig, mlp) -> PartSpec:
    if mlp is None:
        return PartSpec("none", {})
    if mlp["kind"] == "dense":
        return PartSpec("gated", dict(width=cfg.width, inner=mlp["ff"], activation="clamped_swiglu", limit=mlp["limit"],
                                      names=("gate", "up", "down")))
    r = mlp["router"]
    return PartSpec("mixture", dict(
        width=cfg.width, experts=r["experts"], top=r["top"], inner=mlp["expert"]["ff"], score="softmax", renormalize=False,
        weight_on="output", activation="silu", router_name="router", correction_name="correction",
        identity=r.get("identity", 0), groups=r.get("groups"), expert_name="e{}.", names=("gate", "up", "down")))


def gubulorn_spec(cfg: GubulornConfig) -> ModelSpec:
    d = cfg.width
    norm = PartSpec("rms_norm", dict(width=d, eps=cfg.eps, weight_suffix="", unit_offset=True))
    no_norm = PartSpec("layer_norm", dict(width=d, eps=cfg.eps, affine=False))       # behind a feed-forward that is not there
    layers, unread = [], []
    for i, layer in enumerate(cfg.layers):
        mlp = layer.get("mlp")
        if mlp is None:
            unread.append(f"l{i}.norm2")
        layers.append(LayerSpec(prefix=f"l{i}.", block=PartSpec("post_norm", dict(alpha=cfg.postln_alpha)),
                                mixer=_mixer(cfg, layer["type"], layer["mixer"]), feed_forward=_feed_forward(cfg, mlp),
                                mixer_norm=norm, feed_forward_norm=norm if mlp is not None else no_norm, mixer_name="mix.",
                                feed_forward_name="mlp.", mixer_norm_name="norm1", feed_forward_norm_name="norm2"))
    embedding = PartSpec("token_table", dict(vocab=cfg.vocab, embed_width=d, width=d, position=PartSpec("none", {}),
                                             table_name="embed", projection_name=None, position_name=None, norm=norm,
                                             norm_name="embed.norm"))
    head = PartSpec("vocab_projection", dict(vocab=cfg.vocab, embed_width=d, width=d, norm=norm, weight_name="head",
                                             tied_to=None, projection_name=None, norm_name="final.norm",
                                             logit_scale=cfg.logit_scale, softcap=cfg.logit_softcap))
    return ModelSpec(hidden_size=d, vocab_size=cfg.vocab, max_positions=cfg.max_positions, embedding=embedding,
                     layers=tuple(layers), schedule=ModelSpec.sequential(len(layers)), head=head,
                     init_std=cfg.init_std, unread=tuple(unread))


ARCHITECTURE = register_architecture("Gubulorn", "gubulorn", GubulornConfig, gubulorn_spec,
                                     model_class="transformers_neuronx_amd.gubulorn.model:GubulornForSampling")
