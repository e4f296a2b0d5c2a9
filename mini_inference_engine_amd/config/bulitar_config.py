"""Configuration of the Bulitar decoder, read from its own ``config.json`` keys.

The file lists the layers one by one; each entry names its mixer kind, the mixer's sizes and constants and its feed-forward.
Mixers: ``attention`` (grouped-query softmax attention within chunks of ``mask.size`` positions, biased projections through a
short convolution, adjacent pairs turned by angles that ``rot.scaling`` may stretch) and ``channel_delta`` (a gated delta rule
whose state decays key channel by key channel).  The feed-forward is a mixture of gated experts (``moe``) or none.  ``loop``
names a stretch of layers that runs several times in a row with the same weights.  Every size and constant that may differ
between two models of the design is a field here.  Two sizes are in no key of the file, the inner sizes of the two low-rank
products of a ``channel_delta`` mixer: they are read from the shapes of the checkpoint's tensors (``reads_tensor_shapes``), or
from the keys ``decay_rank`` and ``gate_rank`` that this reader's own ``to_dict`` writes beside the other sizes.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Mapping

from .model_config import ConfigError, ModelConfig, _take_float, _take_int
from .pokulorn_config import YarnRotarySpec
from .vezodra_config import LoopSpec, _heads
from .zifelorn_config import _section


@dataclass(frozen=True)
class ChunkedAttentionSpec:
    """A query sees the earlier keys of its own chunk of ``chunk`` positions (None: all of them); ``taps`` of the convolution on
    the projections (None: there is none); ``rot`` None: positions do not enter."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rot: YarnRotarySpec | None
    taps: int | None
    chunk: int | None = None
    kind = "attention"

    @classmethod
    def from_dict(cls, d, where, shapes=None, layer=0):
        heads, kv_heads = _heads(d, where)
        dim = _take_int(d, "dim")
        mask = d.get("mask")
        return cls(heads, kv_heads, dim, _take_int(d, "vdim", default=dim), _take_float(d, "scale"),
                   None if d.get("rot") is None else YarnRotarySpec.from_dict(_section(d, "rot", where), where, dim),
                   None if d.get("conv") is None else _take_int(d, "conv"),
                   None if mask is None else _take_int(_section(d, "mask", where), "size"))

    def to_dict(self):
        d = dict(heads=self.heads, kv_heads=self.kv_heads, dim=self.dim, vdim=self.vdim, scale=self.scale)
        if self.rot is not None:
            d["rot"] = self.rot.to_dict()
        if self.taps is not None:
            d["conv"] = self.taps
        if self.chunk is not None:
            d["mask"] = dict(size=self.chunk)
        return d


@dataclass(frozen=True)
class ChannelDeltaSpec:
    """``heads`` states of dim x vdim, queries and keys shared by heads / kv_heads of them; ``decay_rank`` and ``gate_rank`` are the
    inner sizes of the decays' and the output gate's products."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    taps: int | None
    decay_rank: int
    gate_rank: int
    kind = "channel_delta"

    @classmethod
    def from_dict(cls, d, where, shapes=None, layer=0):
        heads, kv_heads = _heads(d, where)
        dim = _take_int(d, "dim")
        ranks = []
        for key, tensor in (("decay_rank", "a1"), ("gate_rank", "g1")):
            rank, name = d.get(key), f"l{layer}.mix.{tensor}"
            if rank is None and shapes is not None and name in shapes:
                rank = int(shapes[name][0])
            if rank is None:
                raise ConfigError(f"config.json: {where}{key} is not given and no checkpoint tensor {name} to read it from")
            if isinstance(rank, bool) or not isinstance(rank, int) or rank < 1:
                raise ConfigError(f"config.json: {where}{key} must be a positive integer, found {rank!r}")
            ranks.append(rank)
        return cls(heads, kv_heads, dim, _take_int(d, "vdim", default=dim), None if d.get("conv") is None else _take_int(d, "conv"), *ranks)

    def to_dict(self):
        d = dict(heads=self.heads, kv_heads=self.kv_heads, dim=self.dim, vdim=self.vdim, decay_rank=self.decay_rank, gate_rank=self.gate_rank)
        if self.taps is not None:
            d["conv"] = self.taps
        return d


@dataclass(frozen=True)
class SigmoidMoESpec:
    """``experts`` gated units of inner size ``expert_ff``, of which a token runs ``top``; the chosen ones' sigmoid scores times
    ``scale`` are their weights."""
    experts: int
    top: int
    expert_ff: int
    scale: float
    kind = "moe"

    @classmethod
    def from_dict(cls, d, where):
        router, expert = _section(d, "router", where), _section(d, "expert", where)
        spec = cls(_take_int(router, "experts"), _take_int(router, "top"), _take_int(expert, "ff"), _take_float(router, "scale", default=1.0))
        if spec.top > spec.experts:
            raise ConfigError(f"config.json: {where}router.top {spec.top} of {spec.experts} experts")
        return spec

    def to_dict(self):
        return dict(kind="moe", expert=dict(ff=self.expert_ff), router=dict(experts=self.experts, top=self.top, scale=self.scale))


_MIXERS = {"attention": ChunkedAttentionSpec, "channel_delta": ChannelDeltaSpec}


@dataclass(frozen=True)
class BulitarLayer:
    mixer: Any
    mlp: Any

    def to_dict(self):
        return dict(type=self.mixer.kind, mixer=self.mixer.to_dict(), mlp=None if self.mlp is None else self.mlp.to_dict())


@dataclass(frozen=True)
class BulitarConfig(ModelConfig):
    vocab: int
    width: int
    layers: tuple
    norm_eps: float
    embedding_scale: float = 1.0
    loop: LoopSpec | None = None

    architecture = "Bulitar"
    reads_tensor_shapes = True          # from_dict takes the checkpoint's tensor shapes beside the dictionary

    def __post_init__(self):
        if not self.layers:
            raise ConfigError("config.json: 'layers' is empty")
        if not self.norm_eps > 0:
            raise ConfigError(f"config.json: norm.eps must be positive, found {self.norm_eps}")
        if self.loop is not None:
            lp = self.loop
            if not 0 <= lp.start < lp.stop <= len(self.layers) or lp.times < 1:
                raise ConfigError(f"config.json: loop {lp.to_dict()} does not name a stretch of the {len(self.layers)} layers")

    def run_order(self) -> list:
        """(layer, pass of the loop that begins right before it, or None) of every layer run."""
        n = len(self.layers)
        if self.loop is None:
            return [(i, None) for i in range(n)]
        lp = self.loop
        passes = [(i, t if i == lp.start else None) for t in range(lp.times) for i in range(lp.start, lp.stop)]
        return [(i, None) for i in range(lp.start)] + passes + [(i, None) for i in range(lp.stop, n)]

    @classmethod
    def from_dict(cls, d: Mapping[str, Any], tensor_shapes=None) -> "BulitarConfig":
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
            mixer = _MIXERS[kind].from_dict(_section(entry, "mixer", where), where + "mixer.", tensor_shapes, i)
            mlp = entry.get("mlp")
            if mlp is not None:
                if not isinstance(mlp, Mapping) or mlp.get("kind") != "moe":
                    raise ConfigError(f"config.json: {where}mlp must be null or of kind 'moe'")
                mlp = SigmoidMoESpec.from_dict(mlp, where + "mlp.")
            layers.append(BulitarLayer(mixer, mlp))
        loop = d.get("loop")
        if loop is not None:
            lp = _section(d, "loop", "")
            loop = LoopSpec(_take_int(lp, "start", minimum=0), _take_int(lp, "stop"), _take_int(lp, "times"))
        emb = d.get("embedding")
        return cls(vocab=_take_int(d, "vocab"), width=_take_int(d, "width"), layers=tuple(layers),
                   norm_eps=_take_float(_section(d, "norm", ""), "eps"),
                   embedding_scale=1.0 if emb is None else _take_float(_section(d, "embedding", ""), "scale", default=1.0), loop=loop)

    def to_dict(self) -> dict:
        d = dict(architecture=self.architecture, vocab=self.vocab, width=self.width, norm=dict(eps=self.norm_eps),
                 embedding=dict(scale=self.embedding_scale), layers=[layer.to_dict() for layer in self.layers])
        if self.loop is not None:
            d["loop"] = self.loop.to_dict()
        return d
