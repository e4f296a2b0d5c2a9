"""Pokulorn: a decoder whose layers are listed one by one in its configuration.

A layer adds its mixer of the normed stream and then its feed-forward of the normed stream; a layer may be its mixer alone.
Mixers: softmax attention with a sink per head under a sliding window that keeps a request's first tokens, its values mixed
with those of the first such layer (``attention``); full attention with an elementwise output gate beside a state space with
one decay a head and step, joined by two fixed factors (``parallel``); matrix memory with exponential gates (``mlstm``).  Both
attentions convolve their projections over the last few tokens, norm queries and keys head by head and turn halves by YaRN
angles.  The feed-forward is a clamped gated unit.  The head has a matrix of its own.  Everything here is construction: sizes
and constants come from PokulornConfig only.
Tensor names: ``embed``, ``head``, ``final.norm``, ``l<i>.norm1|norm2``, ``l<i>.mix.*``, ``l<i>.mlp.*``.
"""
from __future__ import annotations

from ..config.pokulorn_config import ConvAttentionSpec, MatrixMemorySpec, PokulornConfig, ScaledPairSpec
from ..config.registry import register_architecture
from ..parts import (DecoderSpec, Embedding, LMHead, MatrixLSTM, PreNormBlock, RMSNorm, RotaryHalfAngles, RotaryYarn, ScaledPair,
                     SoftmaxAttention, StateSpace, SwiGLU)

GATE_SLOPE, UP_SHIFT = 1.702, 1.0       # of the feed-forward's hidden activation g sigmoid(slope g) (u + shift)


def build_pokulorn(cfg: PokulornConfig) -> DecoderSpec:
    w, eps = cfg.width, cfg.norm_eps
    norm = lambda name: RMSNorm(w, eps, name)        # noqa: E731
    rotations = {}          # one position-encoding part for each distinct rotation

    def rotation(rot):
        if rot not in rotations:
            s = rot.scaling
            rotations[rot] = (RotaryHalfAngles(rot.dims, rot.base) if s is None
                              else RotaryYarn(rot.dims, rot.base, s.factor, s.original, s.fast, s.slow))
        return rotations[rot]

    def attention(m, prefix, **options):
        return SoftmaxAttention(w, m.heads, m.kv_heads, m.dim, m.vdim, m.scale, rotation(m.rot), prefix=prefix, window=m.window,
                                keep_first=m.keep_first, conv=m.taps, qk_norm="head", eps=eps, **options)

    first = cfg.first_value_layer()
    layers = []
    for i, layer in enumerate(cfg.layers):
        m, f, p = layer.mixer, layer.mlp, f"l{i}"
        if isinstance(m, ConvAttentionSpec):
            mixing = {} if not m.v_mix else {"share_values" if i == first else "take_values": "first_values"}
            mixer = attention(m, f"{p}.mix", sink="head", **mixing)
        elif isinstance(m, ScaledPairSpec):
            r = m.right
            mixer = ScaledPair(w, attention(m.left, f"{p}.mix.left", element_gate=True),
                               StateSpace(w, r.heads, r.vdim, r.state, r.groups, r.taps, r.norm_groups, eps, prefix=f"{p}.mix.right"),
                               m.left_scale, m.right_scale)
        elif isinstance(m, MatrixMemorySpec):
            mixer = MatrixLSTM(w, m.heads, m.dim, m.vdim, m.gate_cap, eps, prefix=f"{p}.mix")
        else:
            raise TypeError(f"layer {i}: no part for mixer {m!r}")
        ff = norm2 = None
        if f is not None:
            norm2 = norm(f"{p}.norm2")
            ff = SwiGLU(w, f.ff, prefix=f"{p}.mlp", tensor_names=("gate", "up", "down"), clamp=(f.limit, GATE_SLOPE, UP_SHIFT))
        layers.append(PreNormBlock(norm(f"{p}.norm1"), mixer, norm2, ff))
    return DecoderSpec(embedding=Embedding(cfg.vocab, w, "embed"), layers=layers, final_norm=norm("final.norm"),
                       head=LMHead(cfg.vocab, w, "head"), stop_token_ids=(), max_position=None, vocab_size=cfg.vocab)


def _shape(vocab, width, ff, heads, kv_heads, dim, window, keep_first, pair_heads, pair_kv_heads, pair_dim, ssm_heads, ssm_vdim,
           ssm_state, ssm_groups, mem_heads, mem_dim, mem_vdim, repeats):
    """A named size: ``repeats`` times the run (parallel, attention, mlstm), the last layer of each without a feed-forward in
    every second run."""
    rot = lambda dims: dict(base=10000.0, dims=dims, scaling=dict(factor=4.0, original=2048, fast=32.0, slow=1.0))        # noqa: E731
    att = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=dim, scale=dim ** -0.5, rot=rot(dim), conv=4, v_mix=True,
               mask=dict(size=window, keep_first=keep_first))
    pair = dict(left=dict(heads=pair_heads, kv_heads=pair_kv_heads, dim=pair_dim, vdim=pair_dim, scale=pair_dim ** -0.5,
                          rot=rot(pair_dim // 2), conv=4),
                right=dict(heads=ssm_heads, vdim=ssm_vdim, state=ssm_state, groups=ssm_groups, conv=4, norm_groups=ssm_groups),
                left_scale=0.5, right_scale=0.5)
    mem = dict(heads=mem_heads, dim=mem_dim, vdim=mem_vdim, gate_cap=15.0)
    dense = dict(kind="dense", ff=ff, limit=7.0)
    layers = []
    for r in range(repeats):
        layers += [dict(type="parallel", mixer=pair, mlp=dense), dict(type="attention", mixer=att, mlp=dense),
                   dict(type="mlstm", mixer=mem, mlp=dense if r % 2 == 0 else None)]
    return dict(vocab=vocab, width=width, norm=dict(eps=1e-6), layers=layers)


# Named sizes: one for tests and the command line's examples, one with the widths of a 1B-class model.
SHAPES = {
    "pokulorn-tiny": _shape(vocab=320, width=64, ff=112, heads=4, kv_heads=2, dim=16, window=24, keep_first=3, pair_heads=3,
                            pair_kv_heads=1, pair_dim=32, ssm_heads=4, ssm_vdim=16, ssm_state=24, ssm_groups=2, mem_heads=2,
                            mem_dim=16, mem_vdim=24, repeats=2),
    "pokulorn-1b": _shape(vocab=32000, width=2048, ff=5632, heads=32, kv_heads=8, dim=64, window=1024, keep_first=4, pair_heads=16,
                          pair_kv_heads=4, pair_dim=128, ssm_heads=32, ssm_vdim=64, ssm_state=128, ssm_groups=8, mem_heads=8,
                          mem_dim=128, mem_vdim=256, repeats=5),
}

register_architecture("Pokulorn", PokulornConfig, build_pokulorn, shapes=SHAPES, replace=True)
