"""Configuration of the Narasun decoder, from its config.json.

The file is nested: the model's own sizes and constants at the top (``vocab``, ``width``, ``norm.eps``, ``loop``) and a list
``layers`` whose entries each give the layer's ``type`` (its mixer), the mixer's sizes and constants (``mixer``) and its
feed-forward (``mlp``, or null for a layer without one).  Layers need not be alike: the plan is built layer by layer.

    parallel           two mixers side by side and the factors on their outputs: left_scale, right_scale,
                       left     softmax attention: heads, kv_heads (absent: heads), dim, vdim (absent: dim), scale, q_temp.coef /
                                q_temp.every (the query's factor by position; absent: none)
                       right    time mixing: heads, dim (keys and values alike), rank (the width of the decay's low-rank
                                projection; a file that leaves it out leaves it to the tensor's shape)
    mlstm, mlstm_2     matrix memory with exponential gates: heads, dim (queries and keys), vdim (absent: dim), gate_cap
    mlp                kind "dense": ff
                       kind "moe": expert.ff, router.experts / top
    loop               start, stop, times: layers start .. stop - 1 run ``times`` times in a row with the same weights

A missing or mistyped key is an error that names it by its path.
"""
from __future__ import annotations

import dataclasses
from typing import Any, ClassVar, Dict, Mapping, Optional, Tuple, Union

from .base import ConfigError, ModelConfig, read_key
from .mumusun import _read, _section
from .tabatar import DenseMlpConfig, LoopConfig, MoeMlpConfig, _mlp_from_dict, run_order_with_passes
from .vavadra import _positive

MATRIX_MEMORY_TYPES = ("mlstm", "mlstm_2")
MIXER_TYPES = ("parallel", *MATRIX_MEMORY_TYPES)


@dataclasses.dataclass(frozen=True)
class QueryTemperature:
    coef: float
    every: int

    def to_dict(self) -> Dict[str, Any]:
        return {"coef": self.coef, "every": self.every}


@dataclasses.dataclass(frozen=True)
class SinkAttentionConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    q_temp: Optional[QueryTemperature]

    @classmethod
    def from_dict(cls, d: Mapping[str, Any], where: str) -> "SinkAttentionConfig":
        dim, heads = _read(d, "dim", int, where), _read(d, "heads", int, where)
        temp = _section(d, "q_temp", where, optional=True)
        if temp is not None:
            temp = QueryTemperature(_read(temp, "coef", float, where + "q_temp."), _read(temp, "every", int, where + "q_temp."))
        return cls(heads=heads, kv_heads=_read(d, "kv_heads", int, where, heads), dim=dim, vdim=_read(d, "vdim", int, where, dim),
                   scale=_read(d, "scale", float, where), q_temp=temp)

    def to_dict(self) -> Dict[str, Any]:
        out = {"heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim, "vdim": self.vdim, "scale": self.scale}
        if self.q_temp is not None:
            out["q_temp"] = self.q_temp.to_dict()
        return out

    def validate(self, where: str) -> None:
        _positive(self, ("heads", "kv_heads", "dim", "vdim"), where)
        if self.heads % self.kv_heads:
            raise ConfigError(f"config.json: '{where}heads' = {self.heads} is not a multiple of kv_heads {self.kv_heads}")
        if self.q_temp is not None and self.q_temp.every <= 0:
            raise ConfigError(f"config.json: '{where}q_temp.every' must be positive, got {self.q_temp.every}")


@dataclasses.dataclass(frozen=True)
class TimeMixConfig:
    heads: int
    dim: int
    rank: Optional[int]        # None: the model file's tensors say (``with_tensor_shapes``)

    @classmethod
    def from_dict(cls, d: Mapping[str, Any], where: str) -> "TimeMixConfig":
        return cls(heads=_read(d, "heads", int, where), dim=_read(d, "dim", int, where), rank=_read(d, "rank", int, where, None))

    def to_dict(self) -> Dict[str, Any]:
        out = {"heads": self.heads, "dim": self.dim}
        if self.rank is not None:
            out["rank"] = self.rank
        return out

    def validate(self, where: str) -> None:
        _positive(self, ("heads", "dim"), where)
        if self.rank is not None and self.rank <= 0:
            raise ConfigError(f"config.json: '{where}rank' must be positive, got {self.rank}")


@dataclasses.dataclass(frozen=True)
class ParallelMixersConfig:
    left: SinkAttentionConfig
    right: TimeMixConfig
    left_scale: float
    right_scale: float

    @classmethod
    def from_dict(cls, d: Mapping[str, Any], where: str) -> "ParallelMixersConfig":
        return cls(left=SinkAttentionConfig.from_dict(_section(d, "left", where), where + "left."),
                   right=TimeMixConfig.from_dict(_section(d, "right", where), where + "right."),
                   left_scale=_read(d, "left_scale", float, where), right_scale=_read(d, "right_scale", float, where))

    def to_dict(self) -> Dict[str, Any]:
        return {"left": self.left.to_dict(), "right": self.right.to_dict(), "left_scale": self.left_scale, "right_scale": self.right_scale}

    def validate(self, where: str) -> None:
        self.left.validate(where + "left.")
        self.right.validate(where + "right.")


@dataclasses.dataclass(frozen=True)
class MatrixMemoryConfig:
    heads: int
    dim: int
    vdim: int
    gate_cap: float

    @classmethod
    def from_dict(cls, d: Mapping[str, Any], where: str) -> "MatrixMemoryConfig":
        dim = _read(d, "dim", int, where)
        return cls(heads=_read(d, "heads", int, where), dim=dim, vdim=_read(d, "vdim", int, where, dim),
                   gate_cap=_read(d, "gate_cap", float, where))

    def to_dict(self) -> Dict[str, Any]:
        return {"heads": self.heads, "dim": self.dim, "vdim": self.vdim, "gate_cap": self.gate_cap}

    def validate(self, where: str) -> None:
        _positive(self, ("heads", "dim", "vdim", "gate_cap"), where)


@dataclasses.dataclass(frozen=True)
class NarasunLayer:
    type: str
    mixer: Union[ParallelMixersConfig, MatrixMemoryConfig]
    mlp: Union[None, DenseMlpConfig, MoeMlpConfig]

    def to_dict(self) -> Dict[str, Any]:
        return {"type": self.type, "mixer": self.mixer.to_dict(), "mlp": self.mlp.to_dict() if self.mlp is not None else None}


@dataclasses.dataclass(frozen=True)
class NarasunConfig(ModelConfig):
    vocab: int
    width: int
    norm_eps: float
    loop: Optional[LoopConfig]
    layers: Tuple[NarasunLayer, ...]
    # The file names no longest sequence: positions are formed in 32-bit floats, which count integers exactly up to 2^24.
    max_positions: int = 1 << 24

    model_type: ClassVar[str] = "narasun"
    architectures: ClassVar[Tuple[str, ...]] = ("Narasun",)

    @classmethod
    def from_dict(cls, d: Mapping[str, Any]) -> "NarasunConfig":
        layers_in = d.get("layers")
        if not isinstance(layers_in, list) or not layers_in:
            raise ConfigError("config.json: 'layers' must be a non-empty list")
        layers = []
        for i, L in enumerate(layers_in):
            where = f"layers[{i}]."
            if not isinstance(L, dict):
                raise ConfigError(f"config.json: 'layers[{i}]' must be an object")
            kind = _read(L, "type", str, where)
            if kind not in MIXER_TYPES:
                raise ConfigError(f"config.json: '{where}type' = '{kind}' is not a known mixer (one of {MIXER_TYPES})")
            mixer_cls = ParallelMixersConfig if kind == "parallel" else MatrixMemoryConfig
            mixer = mixer_cls.from_dict(_section(L, "mixer", where), where + "mixer.")
            mlp = _section(L, "mlp", where, optional=True)
            mlp = _mlp_from_dict(mlp, where + "mlp.") if mlp is not None else None
            if getattr(mlp, "shared_ff", 0):
                raise ConfigError(f"config.json: '{where}mlp.shared': the design has no shared expert")
            layers.append(NarasunLayer(kind, mixer, mlp))
        norm = _section(d, "norm", "")
        lp = _section(d, "loop", "", optional=True)
        loop = None
        if lp is not None:
            loop = LoopConfig(_read(lp, "start", int, "loop."), _read(lp, "stop", int, "loop."), _read(lp, "times", int, "loop.", 1))
        cfg = cls(vocab=read_key(d, "vocab", int), width=read_key(d, "width", int), norm_eps=_read(norm, "eps", float, "norm."),
                  loop=loop, layers=tuple(layers), max_positions=read_key(d, "max_positions", int, 1 << 24))
        cfg.validate()
        return cfg

    def to_dict(self) -> Dict[str, Any]:
        out = {"architecture": self.architectures[0], "vocab": self.vocab, "width": self.width, "norm": {"eps": self.norm_eps},
               "layers": [L.to_dict() for L in self.layers]}
        if self.loop is not None:
            out["loop"] = self.loop.to_dict()
        if self.max_positions != 1 << 24:
            out["max_positions"] = self.max_positions
        return out

    def validate(self) -> None:
        _positive(self, ("vocab", "width", "max_positions"), "")
        if not self.norm_eps >= 0:
            raise ConfigError(f"config.json: 'norm.eps' must be >= 0, got {self.norm_eps}")
        if self.loop is not None:
            lp = self.loop
            if not 0 <= lp.start < lp.stop <= len(self.layers):
                raise ConfigError(f"config.json: 'loop' = layers {lp.start} .. {lp.stop} - 1 does not lie within the {len(self.layers)} layers")
            if lp.times <= 0:
                raise ConfigError(f"config.json: 'loop.times' must be positive, got {lp.times}")
        for i, L in enumerate(self.layers):
            L.mixer.validate(f"layers[{i}].mixer.")
            if L.mlp is not None:
                L.mlp.validate(f"layers[{i}].mlp.")

    def run_order(self) -> Tuple[Tuple[int, Optional[int]], ...]:
        """(layer, pass) in the order the layers run (see ``run_order_with_passes``)."""
        return run_order_with_passes(self.loop, len(self.layers))

    def _rank_is_open(self, i: int) -> bool:
        return self.layers[i].type == "parallel" and self.layers[i].mixer.right.rank is None

    def open_sizes(self) -> Tuple[str, ...]:
        return tuple(f"layers[{i}].mixer.right.rank" for i in range(len(self.layers)) if self._rank_is_open(i))

    def with_tensor_shapes(self, shapes: Mapping[str, Tuple[int, ...]]) -> "NarasunConfig":
        """The config with the sizes it leaves open taken from the model file: the rank of a time mixing's decay is the number
        of rows of its ``l<i>.mix.right.w1``."""
        layers = list(self.layers)
        for i, L in enumerate(layers):
            if self._rank_is_open(i):
                shape = shapes.get(f"l{i}.mix.right.w1")
                if shape is None or len(shape) != 2:
                    raise ConfigError(f"config.json: 'layers[{i}].mixer.right' names no rank and the model file has no matrix "
                                      f"'l{i}.mix.right.w1' to take it from")
                right = dataclasses.replace(L.mixer.right, rank=int(shape[0]))
                layers[i] = dataclasses.replace(L, mixer=dataclasses.replace(L.mixer, right=right))
        out = dataclasses.replace(self, layers=tuple(layers))
        out.validate()
        return out
