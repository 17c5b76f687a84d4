"""Typed configuration of the Fuvevik family, read from the keys of its ``config.json``.

Every size and every constant that one model of the design may choose differently from another comes from the
file: ``streams`` and ``layers``, of which each entry gives its ``type`` (which mixer), the mixer's sizes and constants and
its feed-forward (``mlp``; null: the layer has none).  A key the file must give and does not is an error that names it; an
absent ``q_temp``, ``kv_from``, router ``identity`` or ``mlp.shared`` switches its mechanism off.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Dict, Optional, Tuple, Union

from .fusavik_config import _need, _positive
from .model_config import ConfigError

LAYER_TYPES = ("attention",)
MLP_KINDS = ("dense", "moe")


@dataclass(frozen=True)
class TemperedAttentionConfig:
    """Causal softmax attention with grouped heads and no rotation: a norm a head on queries and keys, a query factor that
    grows with the position (``q_temp`` = (coef, every)), a sink in the denominator and a gate a channel.  ``kv_from``: the
    layer whose keys and values this one reads instead of making its own."""

    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    q_temp: Optional[Tuple[float, int]]
    kv_from: Optional[int]

    @staticmethod
    def from_dict(d: Dict[str, Any], where: str) -> "TemperedAttentionConfig":
        temp = d.get("q_temp")
        if temp is not None:
            temp = (float(_need(temp, "coef", where + ".q_temp")), int(_need(temp, "every", where + ".q_temp")))
            _positive(temp[1], f"{where}.q_temp.every")
        out = TemperedAttentionConfig(int(_need(d, "heads", where)), int(_need(d, "kv_heads", where)), int(_need(d, "dim", where)),
                                      int(_need(d, "vdim", where)), float(_need(d, "scale", where)), temp,
                                      None if d.get("kv_from") is None else int(d["kv_from"]))
        for name in ("heads", "kv_heads", "dim", "vdim"):
            _positive(getattr(out, name), f"{where}.{name}")
        if out.heads % out.kv_heads:
            raise ConfigError(f"{where}: {out.heads} heads do not divide into {out.kv_heads} kv heads")
        return out

    def to_dict(self) -> Dict[str, Any]:
        d: Dict[str, Any] = {"dim": self.dim, "heads": self.heads, "kv_heads": self.kv_heads, "scale": self.scale, "vdim": self.vdim}
        if self.q_temp is not None:
            d["q_temp"] = {"coef": self.q_temp[0], "every": self.q_temp[1]}
        if self.kv_from is not None:
            d["kv_from"] = self.kv_from
        return d


@dataclass(frozen=True)
class DenseConfig:
    """A feed-forward without a gate, ``ff`` hidden units."""

    ff: int

    @staticmethod
    def from_dict(d: Dict[str, Any], where: str) -> "DenseConfig":
        return DenseConfig(_positive(int(_need(d, "ff", where)), f"{where}.ff"))

    def to_dict(self) -> Dict[str, Any]:
        return {"ff": self.ff, "kind": "dense"}


@dataclass(frozen=True)
class SharedScoreExpertsConfig:
    """Routed experts with hidden units capped at ``limit``, and ``identity`` more that give their input back: chosen by the
    softmax over all of them plus a correction, weighed by the chosen ones' shares of the softmax over their sum.
    ``shared`` (ff, limit): one more expert every token uses."""

    experts: int
    identity: int
    top: int
    ff: int
    limit: float
    shared: Optional[Tuple[int, float]]

    @staticmethod
    def from_dict(d: Dict[str, Any], where: str) -> "SharedScoreExpertsConfig":
        router, expert, shared = _need(d, "router", where), _need(d, "expert", where), d.get("shared")
        if shared is not None:
            shared = (int(_need(shared, "ff", where + ".shared")), float(_need(shared, "limit", where + ".shared")))
            _positive(shared[0], f"{where}.shared.ff")
            _positive(shared[1], f"{where}.shared.limit")
        out = SharedScoreExpertsConfig(int(_need(router, "experts", where + ".router")), int(router.get("identity") or 0),
                                       int(_need(router, "top", where + ".router")), int(_need(expert, "ff", where + ".expert")),
                                       float(_need(expert, "limit", where + ".expert")), shared)
        for name in ("experts", "top", "ff", "limit"):
            _positive(getattr(out, name), f"{where}.{name}")
        if out.identity < 0:
            raise ConfigError(f"{where}.router.identity must not be negative")
        if out.top > out.experts + out.identity:
            raise ConfigError(f"{where}: {out.top} of {out.experts + out.identity} experts cannot be chosen")
        return out

    def to_dict(self) -> Dict[str, Any]:
        d: Dict[str, Any] = {"expert": {"ff": self.ff, "limit": self.limit}, "kind": "moe",
                             "router": {"experts": self.experts, "identity": self.identity, "top": self.top}}
        if self.shared is not None:
            d["shared"] = {"ff": self.shared[0], "limit": self.shared[1]}
        return d


_MLPS = {"dense": DenseConfig, "moe": SharedScoreExpertsConfig}


@dataclass(frozen=True)
class FuvevikLayer:
    type: str
    mixer: TemperedAttentionConfig
    mlp: Optional[Union[DenseConfig, SharedScoreExpertsConfig]]


@dataclass(frozen=True)
class FuvevikConfig:
    architecture: str
    vocab: int
    width: int
    streams: int
    norm_eps: float
    layers: Tuple[FuvevikLayer, ...]
    torch_dtype: str = "bfloat16"

    @staticmethod
    def from_dict(d: Dict[str, Any]) -> "FuvevikConfig":
        name = d.get("architecture") or (d.get("architectures") or [None])[0]
        if not name:
            raise ConfigError("config.json lacks 'architecture'")
        layers = []
        for i, entry in enumerate(_need(d, "layers", "")):
            where = f"layers[{i}]"
            kind = str(_need(entry, "type", where))
            if kind not in LAYER_TYPES:
                raise ConfigError(f"{where}: layer type {kind!r} is not one of {LAYER_TYPES}")
            mlp = entry.get("mlp")
            if mlp is not None:
                form = str(_need(mlp, "kind", where + ".mlp"))
                if form not in _MLPS:
                    raise ConfigError(f"{where}.mlp.kind {form!r} is not one of {MLP_KINDS}")
                mlp = _MLPS[form].from_dict(mlp, where + ".mlp")
            layers.append(FuvevikLayer(kind, TemperedAttentionConfig.from_dict(_need(entry, "mixer", where), where + ".mixer"), mlp))
        if not layers:
            raise ConfigError("config.json lists no layers")
        for i, layer in enumerate(layers):
            src = layer.mixer.kv_from
            if src is None:
                continue
            where = f"layers[{i}].mixer.kv_from"
            if not 0 <= src < i or layers[src].mixer.kv_from is not None:
                raise ConfigError(f"{where} = {src} does not name an earlier layer with keys and values of its own")
            a, b = layers[src].mixer, layer.mixer
            if (a.kv_heads, a.dim, a.vdim) != (b.kv_heads, b.dim, b.vdim):
                raise ConfigError(f"{where}: layer {src} keeps {a.kv_heads} heads of {a.dim} + {a.vdim} channels, "
                                  f"this layer reads {b.kv_heads} of {b.dim} + {b.vdim}")
        cfg = FuvevikConfig(architecture=str(name), vocab=int(_need(d, "vocab", "")), width=int(_need(d, "width", "")),
                            streams=int(_need(d, "streams", "")), norm_eps=float(_need(_need(d, "norm", ""), "eps", "norm")),
                            layers=tuple(layers), torch_dtype=str(d.get("torch_dtype", "bfloat16")))
        _positive(cfg.vocab, "vocab")
        _positive(cfg.width, "width")
        _positive(cfg.streams, "streams")
        _positive(cfg.norm_eps, "norm.eps")
        return cfg

    def to_dict(self) -> Dict[str, Any]:
        return {"architecture": self.architecture, "vocab": self.vocab, "width": self.width, "streams": self.streams,
                "norm": {"eps": self.norm_eps},
                "layers": [{"type": l.type, "mixer": l.mixer.to_dict(), "mlp": None if l.mlp is None else l.mlp.to_dict()}
                           for l in self.layers]}
