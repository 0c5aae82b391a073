"""Solulix's configuration: a nested config.json.

    {"architecture": "Solulix", "vocab": V, "width": D, "norm": {"eps": e}, "loop"?: {"start", "stop", "times"},
     "layers": [{"type": "attention",
                 "mixer": {"heads", "kv_heads", "dim", "vdim", "conv", "scale", "mask": {"size", "keep_first"}},
                 "mlp": MLP},
                {"type": "delta",
                 "mixer": {"heads", "kv_heads", "dim", "vdim", "conv"},
                 "mlp": MLP}, ...]}
    MLP = null | {"kind": "dense", "ff"} |
          {"kind": "moe", "expert": {"ff"}, "router": {"experts", "identity"?, "scale", "top"}, "shared"?: {"ff"}}

Every size and constant is read from there; the layers may come in any order and number.  `loop`: the layers start ..
stop - 1 run `times` times in a row, each pass with a cache and states of its own.
"""
import dataclasses
from typing import Optional, Tuple, Union

from .base import ConfigError, ModelConfig, _coerce
from .vogunex import _need, _positive


@dataclasses.dataclass(frozen=True)
class ConvAttentionConfig:
    heads: int
    kv_heads: int
    dim: int                 # query/key elements per head
    vdim: int                # value elements per head
    conv: int                # taps of the convolutions on queries, keys and values
    scale: float
    window: int              # positions a query sees, its own included ...
    keep_first: int          # ... beside the sequence's first ones

    @staticmethod
    def from_dict(d, where):
        mask = d.get("mask") if isinstance(d, dict) else None
        m = ConvAttentionConfig(**{k: _need(d, k, "int", where) for k in ("heads", "kv_heads", "dim", "vdim", "conv")},
                                scale=_need(d, "scale", "float", where), window=_need(mask, "size", "int", where + ".mask"),
                                keep_first=_need(mask, "keep_first", "int", where + ".mask"))
        _positive(m, ("heads", "kv_heads", "dim", "vdim", "conv", "scale", "window"), where)
        if m.keep_first < 0:
            raise ConfigError(f"config key '{where}.mask.keep_first' must not be negative, found {m.keep_first}")
        if m.heads % m.kv_heads:
            raise ConfigError(f"'{where}': {m.heads} heads are no multiple of {m.kv_heads} kv_heads")
        return m

    def to_dict(self):
        return {"heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim, "vdim": self.vdim, "conv": self.conv, "scale": self.scale,
                "mask": {"size": self.window, "keep_first": self.keep_first}}


@dataclasses.dataclass(frozen=True)
class DeltaConfig:
    heads: int               # value heads
    kv_heads: int            # query/key heads
    dim: int                 # query/key elements per head
    vdim: int                # value elements per head
    conv: int                # taps of the convolutions on queries, keys and values

    @staticmethod
    def from_dict(d, where):
        m = DeltaConfig(**{k: _need(d, k, "int", where) for k in ("heads", "kv_heads", "dim", "vdim", "conv")})
        _positive(m, ("heads", "kv_heads", "dim", "vdim", "conv"), where)
        if m.heads % m.kv_heads:
            raise ConfigError(f"'{where}': {m.heads} heads are no multiple of {m.kv_heads} kv_heads")
        return m

    def to_dict(self):
        return dataclasses.asdict(self)


@dataclasses.dataclass(frozen=True)
class SolulixFeedForwardConfig:
    kind: str                # "dense" or "moe"
    ff: int                  # width of the dense layer, or of one expert
    experts: int = 0         # experts with matrices
    identity: int = 0        # router outputs that stand for the input itself
    top: int = 0
    router_scale: float = 1.0
    shared_ff: Optional[int] = None

    @staticmethod
    def from_dict(d, where):
        kind = _need(d, "kind", "str", where)
        if kind == "dense":
            f = SolulixFeedForwardConfig("dense", _need(d, "ff", "int", where))
        elif kind == "moe":
            ex, ro, sh = d.get("expert"), d.get("router"), d.get("shared")
            r = where + ".router"
            experts, top, scale = _need(ro, "experts", "int", r), _need(ro, "top", "int", r), _need(ro, "scale", "float", r)
            f = SolulixFeedForwardConfig(
                "moe", _need(ex, "ff", "int", where + ".expert"), experts=experts,
                identity=_coerce(r + ".identity", "opt_int", ro.get("identity")) or 0, top=top, router_scale=scale,
                shared_ff=None if sh is None else _need(sh, "ff", "int", where + ".shared"))
            if f.experts <= 0 or f.identity < 0 or not 0 < f.top <= f.experts + f.identity:
                raise ConfigError(f"'{r}': experts ({f.experts}) must be positive and top ({f.top}) lie between 1 and experts + identity "
                                  f"({f.experts} + {f.identity})")
            if f.shared_ff is not None and f.shared_ff <= 0:
                raise ConfigError(f"'{where}.shared.ff' must be positive, found {f.shared_ff}")
        else:
            raise ConfigError(f"'{where}.kind' is '{kind}': neither dense nor moe")
        if f.ff <= 0:
            raise ConfigError(f"'{where}': ff must be positive, found {f.ff}")
        return f

    def to_dict(self):
        if self.kind == "dense":
            return {"kind": "dense", "ff": self.ff}
        d = {"kind": "moe", "expert": {"ff": self.ff},
             "router": {"experts": self.experts, "identity": self.identity, "scale": self.router_scale, "top": self.top}}
        if self.shared_ff is not None:
            d["shared"] = {"ff": self.shared_ff}
        return d


@dataclasses.dataclass(frozen=True)
class LoopConfig:
    start: int
    stop: int
    times: int

    @staticmethod
    def from_dict(d, layers):
        l = LoopConfig(**{k: _need(d, k, "int", "loop") for k in ("start", "stop", "times")})
        if not 0 <= l.start < l.stop <= layers or l.times < 1:
            raise ConfigError(f"'loop': start ({l.start}) must lie below stop ({l.stop}) inside the {layers} layers, and times ({l.times}) be positive")
        return l


MIXERS = {"attention": ConvAttentionConfig, "delta": DeltaConfig}


@dataclasses.dataclass(frozen=True)
class SolulixLayerConfig:
    type: str
    mixer: Union[ConvAttentionConfig, DeltaConfig]
    mlp: Optional[SolulixFeedForwardConfig]


@dataclasses.dataclass
class SolulixConfig(ModelConfig):
    architecture = "Solulix"

    vocab_size: int = 0
    hidden_size: int = 0
    norm_eps: float = 1e-6
    layers: Tuple[SolulixLayerConfig, ...] = ()
    loop: Optional[LoopConfig] = None

    @classmethod
    def from_dict(cls, d):
        if not isinstance(d, dict):
            raise ConfigError("config.json must hold a JSON object")
        layers = d.get("layers")
        if not isinstance(layers, list):
            raise ConfigError("config.json has no 'layers' list")
        out = []
        for i, l in enumerate(layers):
            where = f"layers[{i}]"
            kind = _need(l, "type", "str", where)
            if kind not in MIXERS:
                raise ConfigError(f"'{where}.type' is '{kind}': this design's mixers are {', '.join(MIXERS)}")
            mlp = l.get("mlp")
            out.append(SolulixLayerConfig(kind, MIXERS[kind].from_dict(l.get("mixer"), where + ".mixer"),
                                          None if mlp is None else SolulixFeedForwardConfig.from_dict(mlp, where + ".mlp")))
        cfg = cls(vocab_size=_need(d, "vocab", "int", ""), hidden_size=_need(d, "width", "int", ""),
                  norm_eps=_need(d.get("norm"), "eps", "float", "norm"), layers=tuple(out),
                  loop=None if d.get("loop") is None else LoopConfig.from_dict(d["loop"], len(out)))
        cfg.validate()
        return cfg

    def to_dict(self):
        d = {"architecture": self.architecture, "vocab": self.vocab_size, "width": self.hidden_size, "norm": {"eps": self.norm_eps},
             "layers": [{"type": l.type, "mixer": l.mixer.to_dict(), "mlp": None if l.mlp is None else l.mlp.to_dict()} for l in self.layers]}
        if self.loop is not None:
            d["loop"] = dataclasses.asdict(self.loop)
        return d

    def validate(self):
        if self.vocab_size <= 0 or self.hidden_size <= 0:
            raise ConfigError(f"vocab ({self.vocab_size}) and width ({self.hidden_size}) must be positive")
        if self.norm_eps <= 0:
            raise ConfigError("norm.eps must be positive")
