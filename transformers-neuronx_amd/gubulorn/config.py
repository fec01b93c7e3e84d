"""Gubulorn's configuration: the keys of its config.json.

The file is nested: `norm.eps`, `postln_alpha`, `logit_scale`, `logit_softcap`, and `layers`, a list with one entry a layer:
`type` ("delta" or "parallel"), `mixer` (delta: `{heads, kv_heads, dim, vdim, conv}`; parallel: `left` `{heads, kv_heads, dim,
vdim, scale, q_temp: {coef, every}}` and `right` `{heads, vdim, state, groups, conv, norm_groups}`) and `mlp`
(`{kind: "dense", ff, limit}`, `{kind: "moe", router: {experts, identity, top, groups: {count, keep}}, expert: {ff}}`, or null
for a layer without a feed-forward). Every size and constant of a model is read from there or from a tensor's shape;
the design's own constants are in the code of its parts.
"""
from dataclasses import dataclass
from typing import Any, ClassVar, Dict, Optional

from ..config.model_config import REQUIRED, ConfigError, ModelConfig

MIXERS = ("delta", "parallel")
MLP_KINDS = ("dense", "moe")


def _need(d, key: str, kind, where: str, positive: bool = True):
    if not isinstance(d, dict) or d.get(key) is None:
        raise ConfigError(f"config.json of Gubulorn: required key '{where}.{key}' is missing")
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


def _divides(d, small: str, large: str, where: str) -> None:
    if small in d and d[large] % _need(d, small, int, where):
        raise ConfigError(f"key '{where}.{large}' ({d[large]}) must be a multiple of {small} ({d[small]})")


@dataclass(frozen=True)
class GubulornConfig(ModelConfig):
    architecture: ClassVar[str] = "Gubulorn"
    model_type: ClassVar[str] = "gubulorn"

    vocab: int = REQUIRED
    width: int = REQUIRED
    layers: list = REQUIRED
    norm: dict = REQUIRED
    postln_alpha: float = REQUIRED
    logit_scale: float = 1.0
    logit_softcap: Optional[float] = None
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
        if f.name == "logit_softcap":
            if isinstance(value, bool) or not isinstance(value, (int, float)):
                raise ConfigError(f"key 'logit_softcap' must be a number, got {value!r}")
            return float(value)
        return ModelConfig._coerce(f, value)

    # ---------------------------------------------------------------- what the nested keys say

    @property
    def eps(self) -> float:
        return float(self.norm["eps"])

    def _check_mixer(self, layer, where: str) -> None:
        m, at = layer.get("mixer"), where + ".mixer"
        if layer["type"] == "delta":
            for key in ("heads", "dim", "vdim", "conv"):
                _need(m, key, int, at)
            _divides(m, "kv_heads", "heads", at)
            return
        if not isinstance(m, dict):
            raise ConfigError(f"config.json of Gubulorn: required key '{at}' is missing")
        a, s = m.get("left"), m.get("right")
        for key in ("heads", "dim", "vdim"):
            _need(a, key, int, at + ".left")
        _need(a, "scale", float, at + ".left")
        _divides(a, "kv_heads", "heads", at + ".left")
        if a.get("q_temp") is not None:
            _need(a["q_temp"], "coef", float, at + ".left.q_temp", positive=False)
            _need(a["q_temp"], "every", int, at + ".left.q_temp")
        for key in ("heads", "vdim", "state", "groups", "conv", "norm_groups"):
            _need(s, key, int, at + ".right")
        _divides(s, "groups", "heads", at + ".right")
        if (s["heads"] * s["vdim"]) % s["norm_groups"]:
            raise ConfigError(f"key '{at}.right.norm_groups' ({s['norm_groups']}) must divide heads * vdim "
                              f"({s['heads'] * s['vdim']})")

    def _check_mlp(self, mlp, at: str) -> None:
        if not isinstance(mlp, dict) or mlp.get("kind") not in MLP_KINDS:
            raise ConfigError(f"key '{at}.kind' must be one of {MLP_KINDS}")
        if mlp["kind"] == "dense":
            _need(mlp, "ff", int, at)
            _need(mlp, "limit", float, at)
            return
        r = mlp.get("router")
        total = _need(r, "experts", int, at + ".router")
        top = _need(r, "top", int, at + ".router")
        if r.get("identity") is not None:
            identity = _need(r, "identity", int, at + ".router", positive=False)
            if identity < 0:
                raise ConfigError(f"key '{at}.router.identity' must not be negative, got {identity}")
            total += identity
        chosen_from = total
        if r.get("groups") is not None:
            count = _need(r["groups"], "count", int, at + ".router.groups")
            keep = _need(r["groups"], "keep", int, at + ".router.groups")
            if total % count or keep > count:
                raise ConfigError(f"key '{at}.router.groups': {total} experts in {count} equal groups, {keep} kept")
            chosen_from = keep * (total // count)
        if top > chosen_from:
            raise ConfigError(f"key '{at}.router.top' ({top}) exceeds the {chosen_from} experts that can be chosen")
        _need(mlp.get("expert"), "ff", int, at + ".expert")

    def validate(self) -> None:
        for key in ("vocab", "width", "max_positions"):
            if getattr(self, key) <= 0:
                raise ConfigError(f"key '{key}' must be positive, got {getattr(self, key)}")
        if self.logit_softcap is not None and not self.logit_softcap > 0:
            raise ConfigError(f"key 'logit_softcap' must be positive, got {self.logit_softcap!r}")
        _need(self.norm, "eps", float, "norm")
        for i, layer in enumerate(self.layers):
            where = f"layers[{i}]"
            if not isinstance(layer, dict):
                raise ConfigError(f"key '{where}' must be an object")
            if layer.get("type") not in MIXERS:
                raise ConfigError(f"key '{where}.type' must be one of {MIXERS}, got {layer.get('type')!r}")
            self._check_mixer(layer, where)
            if layer.get("mlp") is not None:
                self._check_mlp(layer["mlp"], where + ".mlp")

    def to_dict(self) -> Dict[str, Any]:
        d = super().to_dict()
        d["architecture"] = self.architecture
        d["model_type"] = self.model_type
        return {k: v for k, v in d.items() if v is not None}
