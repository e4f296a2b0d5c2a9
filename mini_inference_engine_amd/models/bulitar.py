"""Bulitar: a decoder whose layers are listed one by one in its configuration, a stretch of them run several times in a row with
the same weights.

A layer adds its mixer of the normed stream and then its feed-forward of the normed stream; norms are layer norms with a weight
alone.  Mixers: softmax attention within chunks of positions, with biased projections through a short convolution, adjacent pairs
turned by YaRN angles and queries and keys over their root mean square after that (``attention``); a gated delta rule with a decay
per key channel (``channel_delta``).  The feed-forward is a sum of gated experts chosen by sigmoid scores, or absent.  Before each
pass of the loop the stream becomes a product of itself and the embedding's output, plus a vector of the pass.  The embedding is
scaled; the head has a matrix of its own.  Everything here is construction: sizes and constants come from BulitarConfig only.
Tensor names: ``embed``, ``head``, ``final.norm``, ``loop.in``, ``loop.step``, ``l<i>.norm1|norm2``, ``l<i>.mix.*``, ``l<i>.mlp.*``.
"""
from __future__ import annotations

from ..config.bulitar_config import BulitarConfig, ChannelDeltaSpec, ChunkedAttentionSpec
from ..config.registry import register_architecture
from ..parts import (DecoderSpec, Embedding, GatedDelta, LayerCall, LayerNorm, LMHead, LoopEntry, PreNormBlock, RotaryInterleaved,
                     RotaryYarn, RoutedExperts, SoftmaxAttention)


def build_bulitar(cfg: BulitarConfig) -> DecoderSpec:
    w, eps = cfg.width, cfg.norm_eps
    norm = lambda name: LayerNorm(w, eps, name, has_bias=False)        # noqa: E731
    rotations = {None: None}        # one position-encoding part for each distinct rotation

    def rotation(rot):
        if rot not in rotations:
            s = rot.scaling
            rotations[rot] = (RotaryInterleaved(rot.dims, rot.base) if s is None
                              else RotaryYarn(rot.dims, rot.base, s.factor, s.original, s.fast, s.slow, layout="interleaved"))
        return rotations[rot]

    layers = []
    for i, layer in enumerate(cfg.layers):
        m, f, p = layer.mixer, layer.mlp, f"l{i}"
        if isinstance(m, ChunkedAttentionSpec):
            mixer = SoftmaxAttention(w, m.heads, m.kv_heads, m.dim, m.vdim, m.scale, rotation(m.rot), prefix=f"{p}.mix", chunk=m.chunk,
                                     conv=m.taps, qk_norm="turned", eps=eps, bias=True, out_bias=True)
        elif isinstance(m, ChannelDeltaSpec):
            mixer = GatedDelta(w, m.heads, m.kv_heads, m.dim, m.vdim, m.taps, m.decay_rank, m.gate_rank, eps, prefix=f"{p}.mix")
        else:
            raise TypeError(f"layer {i}: no part for mixer {m!r}")
        ff = norm2 = None
        if f is not None:
            norm2 = norm(f"{p}.norm2")
            ff = RoutedExperts(w, f.expert_ff, f.experts, f.top, prefix=f"{p}.mlp", router_bias=False, shares_over="sigmoid",
                               choice_bias=True, gated="silu", share_scale=f.scale)
        layers.append(PreNormBlock(norm(f"{p}.norm1"), mixer, norm2, ff))
    entry = None if cfg.loop is None else LoopEntry(w, cfg.loop.times, "loop.in", "loop.step")
    return DecoderSpec(embedding=Embedding(cfg.vocab, w, "embed", scale=cfg.embedding_scale), layers=layers, final_norm=norm("final.norm"),
                       head=LMHead(cfg.vocab, w, "head"),
                       schedule=[LayerCall(i) if t is None else LayerCall(i, entry=entry, turn=t) for i, t in cfg.run_order()],
                       stop_token_ids=(), max_position=None, vocab_size=cfg.vocab)


def _shape(vocab, width, heads, kv_heads, dim, chunk, delta_heads, delta_kv_heads, delta_dim, delta_vdim, rank, experts, top, expert_ff,
           repeats, times):
    """A named size: ``repeats`` times the run (delta rule, attention, attention), the second layer of the first run looped
    ``times`` times with the third."""
    rot = dict(base=10000.0, dims=dim // 2, scaling=dict(factor=4.0, original=4096, fast=32.0, slow=1.0))
    att = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=dim, scale=dim ** -0.5, conv=4, mask=dict(size=chunk), rot=rot)
    delta = dict(heads=delta_heads, kv_heads=delta_kv_heads, dim=delta_dim, vdim=delta_vdim, conv=4, decay_rank=rank, gate_rank=rank)
    moe = dict(kind="moe", expert=dict(ff=expert_ff), router=dict(experts=experts, top=top, scale=2.0))
    layers = []
    for _ in range(repeats):
        layers += [dict(type="channel_delta", mixer=delta, mlp=moe), dict(type="attention", mixer=att, mlp=moe),
                   dict(type="attention", mixer=att, mlp=moe)]
    return dict(vocab=vocab, width=width, norm=dict(eps=1e-6), embedding=dict(scale=width ** 0.5), loop=dict(start=1, stop=3, times=times),
                layers=layers)


# Named sizes: one for tests and the command line's examples, one with the widths of a 1B-class model.
SHAPES = {
    "bulitar-tiny": _shape(vocab=320, width=64, heads=4, kv_heads=2, dim=16, chunk=24, delta_heads=4, delta_kv_heads=2, delta_dim=16,
                           delta_vdim=24, rank=12, experts=6, top=2, expert_ff=48, repeats=1, times=2),
    "bulitar-1b": _shape(vocab=32000, width=2048, heads=32, kv_heads=4, dim=64, chunk=1024, delta_heads=16, delta_kv_heads=16, delta_dim=128,
                         delta_vdim=128, rank=128, experts=16, top=4, expert_ff=1408, repeats=5, times=2),
}

register_architecture("Bulitar", BulitarConfig, build_bulitar, shapes=SHAPES, replace=True)
