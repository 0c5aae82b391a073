"""Kaderax's configuration: a nested config.json.

    {"architecture": "Kaderax", "vocab": V, "width": D, "norm": {"eps": e}, "residual_mult": m, "loop"?: {"start", "stop", "times"},
     "layers": [{"type": "latent_attention",
                 "mixer": {"heads", "dim", "rot_dim", "vdim", "kv_rank", "q_rank", "scale", "rot": {"base", "dims"}},
                 "mlp": MLP},
                {"type": "parallel",
                 "mixer": {"left": {"heads", "kv_heads", "dim", "vdim", "scale", "softcap", "bias_max", "q_temp": {"coef", "every"}},
                           "left_scale", "right": {"heads", "dim", "vdim", "decay": [g, ...]}, "right_scale"},
                 "mlp": MLP}, ...]}
    MLP = null | {"kind": "dense", "ff"}

Every size and constant is read from there; the layers may come in any order and number.  `loop`: the layers start ..
stop - 1 run `times` times in a row, each pass with a cache and states of its own.
"""
import dataclasses
from typing import Optional, Tuple, Union

from .base import ConfigError, ModelConfig
from .solulix import LoopConfig
from .vogunex import _need, _positive, _rotation


@dataclasses.dataclass(frozen=True)
class BiasedAttentionConfig:
    heads: int
    kv_heads: int
    dim: int                 # query/key elements per head
    vdim: int                # value elements per head
    scale: float
    softcap: float
    bias_max: int            # the distance from which on every key gets the last bias
    temp_coef: float         # the queries' temperature: 1 + coef ln(floor((p + 1) / every) + 1)
    temp_every: int

    @staticmethod
    def from_dict(d, where):
        temp = d.get("q_temp") if isinstance(d, dict) else None
        m = BiasedAttentionConfig(**{k: _need(d, k, "int", where) for k in ("heads", "kv_heads", "dim", "vdim", "bias_max")},
                                  scale=_need(d, "scale", "float", where), softcap=_need(d, "softcap", "float", where),
                                  temp_coef=_need(temp, "coef", "float", where + ".q_temp"), temp_every=_need(temp, "every", "int", where + ".q_temp"))
        _positive(m, ("heads", "kv_heads", "dim", "vdim", "scale", "softcap", "bias_max"), where)
        if m.temp_every <= 0:
            raise ConfigError(f"config key '{where}.q_temp.every' must be positive, found {m.temp_every}")
        if m.heads % m.kv_heads:
            raise ConfigError(f"'{where}': {m.heads} heads are no multiple of {m.kv_heads} kv_heads")
        return m

    def to_dict(self):
        return {"bias_max": self.bias_max, "dim": self.dim, "heads": self.heads, "kv_heads": self.kv_heads,
                "q_temp": {"coef": self.temp_coef, "every": self.temp_every}, "scale": self.scale, "softcap": self.softcap, "vdim": self.vdim}


@dataclasses.dataclass(frozen=True)
class LinearAttentionConfig:
    heads: int
    dim: int                 # query/key elements per head
    vdim: int                # value elements per head
    decay: Tuple[float, ...]

    @staticmethod
    def from_dict(d, where):
        m = LinearAttentionConfig(*(_need(d, k, "int", where) for k in ("heads", "dim", "vdim")), decay=())
        _positive(m, ("heads", "dim", "vdim"), where)
        decay = d.get("decay")
        if not isinstance(decay, list) or len(decay) != m.heads or not all(isinstance(g, (int, float)) and not isinstance(g, bool) and 0 <= g <= 1 for g in decay):
            raise ConfigError(f"config key '{where}.decay' must be a list of {m.heads} numbers between 0 and 1, found {decay!r}")
        return dataclasses.replace(m, decay=tuple(float(g) for g in decay))

    def to_dict(self):
        return {"decay": list(self.decay), "dim": self.dim, "heads": self.heads, "vdim": self.vdim}


@dataclasses.dataclass(frozen=True)
class KaderaxParallelConfig:
    left: BiasedAttentionConfig
    right: LinearAttentionConfig
    left_scale: float
    right_scale: float

    @staticmethod
    def from_dict(d, where):
        if not isinstance(d, dict):
            raise ConfigError(f"config.json: '{where}' must be an object")
        return KaderaxParallelConfig(BiasedAttentionConfig.from_dict(d.get("left"), where + ".left"),
                                     LinearAttentionConfig.from_dict(d.get("right"), where + ".right"),
                                     _need(d, "left_scale", "float", where), _need(d, "right_scale", "float", where))

    def to_dict(self):
        return {"left": self.left.to_dict(), "left_scale": self.left_scale, "right": self.right.to_dict(), "right_scale": self.right_scale}


@dataclasses.dataclass(frozen=True)
class SinkLatentConfig:
    heads: int
    dim: int                 # unrotated query/key elements per head
    rot_dim: int             # rotated query elements per head, and the shared key part's
    vdim: int                # value elements per head
    kv_rank: int             # size of the cached latent
    q_rank: int              # size of the queries' latent
    scale: float
    rot_base: float
    rot_dims: int

    @staticmethod
    def from_dict(d, where):
        m = SinkLatentConfig(**{k: _need(d, k, "int", where) for k in ("heads", "dim", "rot_dim", "vdim", "kv_rank", "q_rank")},
                             scale=_need(d, "scale", "float", where), rot_base=0.0, rot_dims=0)
        _positive(m, ("heads", "dim", "rot_dim", "vdim", "kv_rank", "q_rank", "scale"), where)
        base, dims = _rotation(d, where, m.rot_dim)
        return dataclasses.replace(m, rot_base=base, rot_dims=dims)

    def to_dict(self):
        return {"dim": self.dim, "heads": self.heads, "kv_rank": self.kv_rank, "q_rank": self.q_rank,
                "rot": {"base": self.rot_base, "dims": self.rot_dims}, "rot_dim": self.rot_dim, "scale": self.scale, "vdim": self.vdim}


@dataclasses.dataclass(frozen=True)
class KaderaxFeedForwardConfig:
    ff: int

    @staticmethod
    def from_dict(d, where):
        kind = _need(d, "kind", "str", where)
        if kind != "dense":
            raise ConfigError(f"'{where}.kind' is '{kind}': this design's feed-forward is dense")
        f = KaderaxFeedForwardConfig(_need(d, "ff", "int", where))
        _positive(f, ("ff",), where)
        return f

    def to_dict(self):
        return {"ff": self.ff, "kind": "dense"}


MIXERS = {"latent_attention": SinkLatentConfig, "parallel": KaderaxParallelConfig}


@dataclasses.dataclass(frozen=True)
class KaderaxLayerConfig:
    type: str
    mixer: Union[SinkLatentConfig, KaderaxParallelConfig]
    mlp: Optional[KaderaxFeedForwardConfig]


@dataclasses.dataclass
class KaderaxConfig(ModelConfig):
    architecture = "Kaderax"

    vocab_size: int = 0
    hidden_size: int = 0
    norm_eps: float = 1e-6
    residual_mult: float = 1.0
    layers: Tuple[KaderaxLayerConfig, ...] = ()
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
            out.append(KaderaxLayerConfig(kind, MIXERS[kind].from_dict(l.get("mixer"), where + ".mixer"),
                                          None if mlp is None else KaderaxFeedForwardConfig.from_dict(mlp, where + ".mlp")))
        cfg = cls(vocab_size=_need(d, "vocab", "int", ""), hidden_size=_need(d, "width", "int", ""),
                  norm_eps=_need(d.get("norm"), "eps", "float", "norm"), residual_mult=_need(d, "residual_mult", "float", ""), layers=tuple(out),
                  loop=None if d.get("loop") is None else LoopConfig.from_dict(d["loop"], len(out)))
        cfg.validate()
        return cfg

    def to_dict(self):
        d = {"architecture": self.architecture, "vocab": self.vocab_size, "width": self.hidden_size, "norm": {"eps": self.norm_eps},
             "residual_mult": self.residual_mult,
             "layers": [{"type": l.type, "mixer": l.mixer.to_dict(), "mlp": None if l.mlp is None else l.mlp.to_dict()} for l in self.layers]}
        if self.loop is not None:
            d["loop"] = dataclasses.asdict(self.loop)
        return d

    def validate(self):
        if self.vocab_size <= 0 or self.hidden_size <= 0:
            raise ConfigError(f"vocab ({self.vocab_size}) and width ({self.hidden_size}) must be positive")
        if self.norm_eps <= 0:
            raise ConfigError("norm.eps must be positive")
