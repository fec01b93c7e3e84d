"""Zudusun's configuration: the keys of its config.json.

The file is nested: `norm.eps`, and `layers`, a list with one entry a layer: `type` ("parallel", "attention" or "retention"),
`mixer` (parallel: `left` `{heads, kv_heads, dim, vdim, scale}`, `right` `{heads, dim, vdim, tau}`, `left_scale`,
`right_scale`; attention: `{heads, kv_heads, dim, vdim, scale, rot: {base, dims}, mask: {size}}`; retention: `{heads, dim,
vdim, decay: a list, rot: {base, dims}}`), `mlp` (`{kind: "moe", router: {experts, top}, expert: {ff}, shared: {ff}}`, or
null for a layer without a feed-forward), and `weights_of` where the layer runs with another layer's tensors. Every size
and constant of a model is read from there or from a tensor's shape; the design's own constants are in the code of its
parts.
"""
from dataclasses import dataclass
from typing import Any, ClassVar, Dict

from ..config.model_config import REQUIRED, ConfigError, ModelConfig

MIXERS = ("parallel", "attention", "retention")
MLP_KINDS = ("moe",)


def _need(d, key: str, kind, where: str, positive: bool = True):
    if not isinstance(d, dict) or d.get(key) is None:
        raise ConfigError(f"config.json of Zudusun: required key '{where}.{key}' is missing")
    v = d[key]
    if kind is int and (isinstance(v, bool) or not isinstance(v, int)):
        raise ConfigError(f"key '{where}.{key}' must be an integer, got {v!r}")
    if kind is float:
        if isinstance(v, bool) or not isinstance(v, (int, float)):
            raise ConfigError(f"key '{where}.{key}' must be a number, got {v!r}")
        v = float(v)
    if positive and not v > 0:
        raise ConfigError(f"key '{where}.{key}' must be positive, got {v!r}")
    return v


def _attention_sizes(m, where: str) -> None:
    for key in ("heads", "dim", "vdim"):
        _need(m, key, int, where)
    _need(m, "scale", float, where, positive=False)
    if m.get("kv_heads") is not None and m["heads"] % _need(m, "kv_heads", int, where):
        raise ConfigError(f"key '{where}.heads' ({m['heads']}) must be a multiple of kv_heads ({m['kv_heads']})")


def _rotation(m, where: str) -> None:
    rot = m.get("rot")
    if rot is None:
        return
    _need(rot, "base", float, where + ".rot")
    dims = _need(rot, "dims", int, where + ".rot", positive=False) if rot.get("dims") is not None else m["dim"]
    if dims < 0 or dims % 2 or dims > m["dim"]:
        raise ConfigError(f"key '{where}.rot.dims' ({dims}) must be even and at most dim ({m['dim']})")


@dataclass(frozen=True)
class ZudusunConfig(ModelConfig):
    architecture: ClassVar[str] = "Zudusun"
    model_type: ClassVar[str] = "zudusun"

    vocab: int = REQUIRED
    width: int = REQUIRED
    layers: list = REQUIRED
    norm: dict = REQUIRED
    # not a key of the design, which has no longest request: the most positions the engine's tables are made for
    max_positions: int = 1 << 17
    init_std: float = 0.05
    torch_dtype: str = "bfloat16"

    @staticmethod
    def _coerce(f, value):
        if f.name == "layers":
            if not isinstance(value, list) or not value:
                raise ConfigError(f"key 'layers' must be a list with one entry a layer, got {type(value).__name__}")
            return value
        if f.name == "norm":
            if not isinstance(value, dict):
                raise ConfigError(f"key 'norm' must be an object, got {value!r}")
            return value
        return ModelConfig._coerce(f, value)

    # ---------------------------------------------------------------- what the nested keys say

    @property
    def eps(self) -> float:
        return float(self.norm["eps"])

    def owner(self, i: int) -> int:
        """The layer whose tensors layer i runs with."""
        while self.layers[i].get("weights_of") is not None:
            i = self.layers[i]["weights_of"]
        return i

    def _check_mixer(self, layer, at: str) -> None:
        m = layer.get("mixer")
        if not isinstance(m, dict):
            raise ConfigError(f"config.json of Zudusun: required key '{at}' is missing")
        if layer["type"] == "parallel":
            _attention_sizes(m.get("left"), at + ".left")
            for key in ("heads", "dim", "vdim"):
                _need(m.get("right"), key, int, at + ".right")
            _need(m["right"], "tau", float, at + ".right")
            if m["right"].get("rank") is not None:      # (a checkpoint's tensors say; random weights need the key)
                _need(m["right"], "rank", int, at + ".right")
            for key in ("left_scale", "right_scale"):
                _need(m, key, float, at, positive=False)
        elif layer["type"] == "attention":
            _attention_sizes(m, at)
            _rotation(m, at)
            if m.get("mask") is not None:
                _need(m["mask"], "size", int, at + ".mask")
        else:
            for key in ("heads", "dim", "vdim"):
                _need(m, key, int, at)
            _rotation(m, at)
            decay = m.get("decay")
            if not isinstance(decay, list) or len(decay) != m["heads"] or any(
                    isinstance(x, bool) or not isinstance(x, (int, float)) or not 0 < x <= 1 for x in decay):
                raise ConfigError(f"key '{at}.decay' must be a list of {m['heads']} numbers above 0 and up to 1, got {decay!r}")

    def _check_mlp(self, mlp, at: str) -> None:
        if not isinstance(mlp, dict) or mlp.get("kind") not in MLP_KINDS:
            raise ConfigError(f"key '{at}.kind' must be one of {MLP_KINDS}")
        experts = _need(mlp.get("router"), "experts", int, at + ".router")
        top = _need(mlp["router"], "top", int, at + ".router")
        if top > experts:
            raise ConfigError(f"key '{at}.router.top' ({top}) exceeds the experts ({experts})")
        _need(mlp.get("expert"), "ff", int, at + ".expert")
        if mlp.get("shared") is not None:
            _need(mlp["shared"], "ff", int, at + ".shared")

    def validate(self) -> None:
        for key in ("vocab", "width", "max_positions"):
            if getattr(self, key) <= 0:
                raise ConfigError(f"key '{key}' must be positive, got {getattr(self, key)}")
        _need(self.norm, "eps", float, "norm")
        for i, layer in enumerate(self.layers):
            where = f"layers[{i}]"
            if not isinstance(layer, dict):
                raise ConfigError(f"key '{where}' must be an object")
            if layer.get("type") not in MIXERS:
                raise ConfigError(f"key '{where}.type' must be one of {MIXERS}, got {layer.get('type')!r}")
            self._check_mixer(layer, where + ".mixer")
            if layer.get("mlp") is not None:
                self._check_mlp(layer["mlp"], where + ".mlp")
            at, passed = i, set()
            while self.layers[at].get("weights_of") is not None:
                passed.add(at)
                j = self.layers[at]["weights_of"]
                if isinstance(j, bool) or not isinstance(j, int) or not 0 <= j < len(self.layers) or j in passed:
                    raise ConfigError(f"key 'layers[{at}].weights_of' must name another layer that has tensors, got {j!r}")
                if not isinstance(self.layers[j], dict) or any(self.layers[j].get(k) != layer.get(k)
                                                               for k in ("type", "mixer", "mlp")):
                    raise ConfigError(f"key '{where}.weights_of': layer {j}, whose tensors it runs with, has another type or "
                                      f"other sizes")
                at = j

    def to_dict(self) -> Dict[str, Any]:
        d = super().to_dict()
        d["architecture"] = self.architecture
        d["model_type"] = self.model_type
        return {k: v for k, v in d.items() if v is not None}
