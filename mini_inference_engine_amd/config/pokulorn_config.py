"""Configuration of the Pokulorn decoder, read from its own ``config.json`` keys.

The file lists the layers one by one; each entry names its mixer kind, the mixer's sizes and constants and its feed-forward.
Mixers: ``attention`` (grouped-query softmax attention with a sink per head, an optional sliding window beside kept first
tokens, ``mask``, and values that may be mixed with those of the first layer that mixes, ``v_mix``), ``parallel`` (full
attention with an elementwise output gate, ``left``, beside a state space with one decay a head and step, ``right``, added
with the factors ``left_scale`` and ``right_scale``), ``mlstm`` (matrix memory with exponential gates, their logarithms capped at
``gate_cap``).  Both attentions share the short convolution on the projections (``conv`` taps), the norm per head and the
rotation (``rot``, YaRN where ``rot.scaling`` is given).  The feed-forward is a clamped gated unit (``dense``) or none.
Every size and constant that may differ between two models of the design is a field here.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Mapping

from .model_config import ConfigError, ModelConfig, _take_bool, _take_float, _take_int
from .vezodra_config import _heads
from .zifelorn_config import _section


@dataclass(frozen=True)
class YarnSpec:
    factor: float
    original: float
    fast: float
    slow: float

    def to_dict(self):
        return dict(factor=self.factor, original=self.original, fast=self.fast, slow=self.slow)


@dataclass(frozen=True)
class YarnRotarySpec:
    """The first ``dims`` numbers of a head turn in pairs (which two are a pair is the design's), pair i by base^(-2i / dims) a
    position, stretched by parts where ``scaling`` is given."""
    base: float
    dims: int
    scaling: YarnSpec | None = None

    @classmethod
    def from_dict(cls, d, where, head_dim):
        scaling = None
        if d.get("scaling") is not None:
            s = _section(d, "scaling", where)
            scaling = YarnSpec(*(_take_float(s, k) for k in ("factor", "original", "fast", "slow")))
            if not all(v > 0 for v in scaling.to_dict().values()):
                raise ConfigError(f"config.json: {where}rot.scaling must hold positive numbers, found {scaling.to_dict()}")
        spec = cls(_take_float(d, "base"), _take_int(d, "dims", minimum=2), scaling)
        if spec.dims % 2 or spec.dims > head_dim:
            raise ConfigError(f"config.json: {where}rot.dims {spec.dims} must be even and at most the head size {head_dim}")
        if not spec.base > 0 or (scaling is not None and spec.base == 1):
            raise ConfigError(f"config.json: {where}rot.base must be positive, and not 1 where it is scaled")
        return spec

    def to_dict(self):
        d = dict(base=self.base, dims=self.dims)
        if self.scaling is not None:
            d["scaling"] = self.scaling.to_dict()
        return d


@dataclass(frozen=True)
class ConvAttentionSpec:
    """``taps`` of the convolution on the projections (None: there is none); a query sees the last ``window`` keys (None: all)
    and the request's ``keep_first`` first ones; ``v_mix``: the layer's values are mixed with those of the first layer
    that says so."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rot: YarnRotarySpec
    taps: int | None
    window: int | None = None
    keep_first: int = 0
    v_mix: bool = False
    kind = "attention"

    @classmethod
    def from_dict(cls, d, where):
        heads, kv_heads = _heads(d, where)
        dim = _take_int(d, "dim")
        window, keep = None, 0
        if d.get("mask") is not None:
            mask = _section(d, "mask", where)
            window, keep = _take_int(mask, "size"), _take_int(mask, "keep_first", default=0, minimum=0)
        return cls(heads, kv_heads, dim, _take_int(d, "vdim", default=dim), _take_float(d, "scale"),
                   YarnRotarySpec.from_dict(_section(d, "rot", where), where, dim),
                   None if d.get("conv") is None else _take_int(d, "conv"), window, keep, _take_bool(d, "v_mix", False))

    def to_dict(self):
        d = dict(heads=self.heads, kv_heads=self.kv_heads, dim=self.dim, vdim=self.vdim, scale=self.scale, rot=self.rot.to_dict())
        if self.taps is not None:
            d["conv"] = self.taps
        if self.window is not None:
            d["mask"] = dict(size=self.window, keep_first=self.keep_first)
        if self.v_mix:
            d["v_mix"] = True
        return d


@dataclass(frozen=True)
class StateSpaceSpec:
    """``heads`` states of state x vdim; B and C in ``groups``; ``taps`` of the convolution; the gated output is normed in
    ``norm_groups`` equal parts."""
    heads: int
    vdim: int
    state: int
    groups: int
    taps: int
    norm_groups: int

    @classmethod
    def from_dict(cls, d, where):
        spec = cls(_take_int(d, "heads"), _take_int(d, "vdim"), _take_int(d, "state"), _take_int(d, "groups", default=1),
                   _take_int(d, "conv"), _take_int(d, "norm_groups", default=1))
        if spec.heads % spec.groups:
            raise ConfigError(f"config.json: {where}heads {spec.heads} is not a multiple of groups {spec.groups}")
        if spec.heads * spec.vdim % spec.norm_groups:
            raise ConfigError(f"config.json: {where}heads * vdim {spec.heads * spec.vdim} is not a multiple of norm_groups {spec.norm_groups}")
        return spec

    def to_dict(self):
        return dict(heads=self.heads, vdim=self.vdim, state=self.state, groups=self.groups, conv=self.taps, norm_groups=self.norm_groups)


@dataclass(frozen=True)
class ScaledPairSpec:
    left: ConvAttentionSpec
    right: StateSpaceSpec
    left_scale: float
    right_scale: float
    kind = "parallel"

    @classmethod
    def from_dict(cls, d, where):
        left = ConvAttentionSpec.from_dict(_section(d, "left", where), where + "left.")
        if left.v_mix:
            raise ConfigError(f"config.json: {where}left.v_mix: values are mixed in layers of type attention only")
        return cls(left, StateSpaceSpec.from_dict(_section(d, "right", where), where + "right."),
                   _take_float(d, "left_scale", default=1.0), _take_float(d, "right_scale", default=1.0))

    def to_dict(self):
        return dict(left=self.left.to_dict(), right=self.right.to_dict(), left_scale=self.left_scale, right_scale=self.right_scale)


@dataclass(frozen=True)
class MatrixMemorySpec:
    """``heads`` memories of dim x vdim; the gates' logarithms pass gate_cap * tanh(. / gate_cap)."""
    heads: int
    dim: int
    vdim: int
    gate_cap: float
    kind = "mlstm"

    @classmethod
    def from_dict(cls, d, where):
        dim = _take_int(d, "dim")
        spec = cls(_take_int(d, "heads"), dim, _take_int(d, "vdim", default=dim), _take_float(d, "gate_cap"))
        if not spec.gate_cap > 0:
            raise ConfigError(f"config.json: {where}gate_cap must be positive, found {spec.gate_cap}")
        return spec

    def to_dict(self):
        return dict(heads=self.heads, dim=self.dim, vdim=self.vdim, gate_cap=self.gate_cap)


@dataclass(frozen=True)
class ClampedFFSpec:
    """Dense gated feed-forward of inner size ``ff`` with gate and up values clamped at ``limit``."""
    ff: int
    limit: float
    kind = "dense"

    def to_dict(self):
        return dict(kind="dense", ff=self.ff, limit=self.limit)


_MIXERS = {"attention": ConvAttentionSpec, "parallel": ScaledPairSpec, "mlstm": MatrixMemorySpec}


@dataclass(frozen=True)
class PokulornLayer:
    mixer: Any
    mlp: Any

    def to_dict(self):
        return dict(type=self.mixer.kind, mixer=self.mixer.to_dict(), mlp=None if self.mlp is None else self.mlp.to_dict())


@dataclass(frozen=True)
class PokulornConfig(ModelConfig):
    vocab: int
    width: int
    layers: tuple
    norm_eps: float

    architecture = "Pokulorn"

    def __post_init__(self):
        if not self.layers:
            raise ConfigError("config.json: 'layers' is empty")
        if not self.norm_eps > 0:
            raise ConfigError(f"config.json: norm.eps must be positive, found {self.norm_eps}")
        mixed = {(m.kv_heads, m.vdim) for m in (layer.mixer for layer in self.layers) if getattr(m, "v_mix", False)}
        if len(mixed) > 1:
            raise ConfigError(f"config.json: layers that mix values have values of different sizes (kv_heads, vdim): {sorted(mixed)}")

    def first_value_layer(self) -> int | None:
        """The first layer whose values later ones mix with theirs."""
        return next((i for i, layer in enumerate(self.layers) if getattr(layer.mixer, "v_mix", False)), None)

    @classmethod
    def from_dict(cls, d: Mapping[str, Any]) -> "PokulornConfig":
        raw = d.get("layers")
        if not isinstance(raw, (list, tuple)):
            raise ConfigError("config.json: 'layers' must be a list")
        layers = []
        for i, entry in enumerate(raw):
            where = f"layers[{i}]."
            if not isinstance(entry, Mapping):
                raise ConfigError(f"config.json: layers[{i}] must be an object")
            kind = entry.get("type")
            if kind not in _MIXERS:
                raise ConfigError(f"config.json: {where}type {kind!r} is not computed here ({sorted(_MIXERS)})")
            mixer = _MIXERS[kind].from_dict(_section(entry, "mixer", where), where + "mixer.")
            mlp = entry.get("mlp")
            if mlp is not None:
                if not isinstance(mlp, Mapping) or mlp.get("kind") != "dense":
                    raise ConfigError(f"config.json: {where}mlp must be null or of kind 'dense'")
                mlp = ClampedFFSpec(_take_int(mlp, "ff"), _take_float(mlp, "limit"))
                if not mlp.limit > 0:
                    raise ConfigError(f"config.json: {where}mlp.limit must be positive, found {mlp.limit}")
            layers.append(PokulornLayer(mixer, mlp))
        return cls(vocab=_take_int(d, "vocab"), width=_take_int(d, "width"), layers=tuple(layers),
                   norm_eps=_take_float(_section(d, "norm", ""), "eps"))

    def to_dict(self) -> dict:
        return dict(architecture=self.architecture, vocab=self.vocab, width=self.width, norm=dict(eps=self.norm_eps),
                    layers=[layer.to_dict() for layer in self.layers])
