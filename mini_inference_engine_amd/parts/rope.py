"""Rotary position encoding, half-split pairing.

inv_freq[j] = theta^(-2j/D); angle[p, j] = p * inv_freq[j], both in 32-bit;
out[j] = x[j] cos - x[j + D/2] sin, out[j + D/2] = x[j + D/2] cos + x[j] sin
(inference_engine/model.py:56-69).  ``rotary_dim`` <= head_dim leaves the
trailing dims of each head unrotated (the reference always rotates all of them).
The tables stay in 32-bit whatever the activation dtype is.
"""
from __future__ import annotations

import math

import torch

from .base import PositionEncoding, register_position_encoding


def rotary_tables(theta: float, rotary_dim: int, max_position: int):
    """cos, sin [max_position, rotary_dim / 2] in float32, by the expression of
    inference_engine/model.py:57-61 (the two halves of its table are equal)."""
    exponent = torch.arange(0, rotary_dim, 2, dtype=torch.int64).float() / rotary_dim
    inv_freq = 1.0 / (theta ** exponent)
    t = torch.arange(max_position, dtype=torch.float32)
    freqs = torch.outer(t, inv_freq)
    return freqs.cos().contiguous(), freqs.sin().contiguous()


@register_position_encoding("rotary_half_split")
class RotaryHalfSplit(PositionEncoding):
    def __init__(self, head_dim: int, theta: float, max_position: int, rotary_dim: int | None = None):
        self.head_dim = int(head_dim)
        self.theta = float(theta)
        self.max_position = int(max_position)
        self.rotary_dim = int(rotary_dim if rotary_dim is not None else head_dim)
        if self.rotary_dim % 2 or not 0 < self.rotary_dim <= self.head_dim:
            raise ValueError(f"rotary_dim {self.rotary_dim} must be even and within head_dim {self.head_dim}")
        self.cos = None
        self.sin = None

    def prepare(self, device, dtype):
        if self.cos is None or self.cos.device != torch.device(device):
            cos, sin = rotary_tables(self.theta, self.rotary_dim, self.max_position)
            self.cos, self.sin = cos.to(device), sin.to(device)

    def encode_and_store(self, ops, qkv, step, num_q_heads, num_kv_heads, k_cache, v_cache, slots):
        """Rotate q and k inside ``qkv`` [T, (Hq + 2 Hkv) D] in place and write k, v to
        their cache slots (inference_engine/model.py:133-134,174-175), in one pass."""
        ops.rotary_kv_store(qkv, step.positions, self.cos, self.sin, self.rotary_dim, num_q_heads,
                            num_kv_heads, self.head_dim, k_cache, v_cache, slots)

    def project_encode_store(self, ops, x, w_qkv, step, num_q_heads, num_kv_heads, k_cache, v_cache, slots):
        """Projection, encoding and cache write together; returns what the backend's paged_attention takes as
        its ``qkv`` (a tensor whose first Hq * D columns are the encoded q, or work the backend has put off
        until then).  The backend may run it as one kernel."""
        return ops.linear_rotary_kv_store(x, w_qkv, step.positions, self.cos, self.sin, self.rotary_dim, num_q_heads,
                                          num_kv_heads, self.head_dim, k_cache, v_cache, slots, for_attention=True)


@register_position_encoding("none")
class NoPosition(PositionEncoding):
    """No encoding: q and k go to attention as projected."""

    def __init__(self, head_dim: int):
        self.head_dim = int(head_dim)

    def encode_and_store(self, ops, qkv, step, num_q_heads, num_kv_heads, k_cache, v_cache, slots):
        ops.rotary_kv_store(qkv, step.positions, None, None, 0, num_q_heads, num_kv_heads, self.head_dim,
                            k_cache, v_cache, slots)

    def project_encode_store(self, ops, x, w_qkv, step, num_q_heads, num_kv_heads, k_cache, v_cache, slots):
        return ops.linear_rotary_kv_store(x, w_qkv, step.positions, None, None, 0, num_q_heads, num_kv_heads,
                                          self.head_dim, k_cache, v_cache, slots, for_attention=True)


@register_position_encoding("rotary_interleaved")
class RotaryInterleaved(PositionEncoding):
    """Adjacent pairs: elements 2i and 2i + 1 of the first ``rotary_dim`` dims turn together by the angle
    position * theta^(-2i / rotary_dim); (u, v) -> (u cos - v sin, v cos + u sin).  The kernels that use it
    compute the angle and its cosine and sine in 32-bit from the position and ``inv_freq`` [rotary_dim / 2]
    themselves, so there is no table and no longest position."""

    layout = "interleaved"
    magnitude = 1.0         # factor on every cosine and sine

    def __init__(self, rotary_dim: int, theta: float, factor: float = 1.0):
        """``factor``: linear scaling, every frequency divided by it."""
        self.rotary_dim = int(rotary_dim)
        self.theta = float(theta)
        self.factor = float(factor)
        if self.rotary_dim % 2 or self.rotary_dim < 2:
            raise ValueError(f"rotary_dim {self.rotary_dim} must be even and at least 2")
        if not self.theta > 0 or not self.factor > 0:
            raise ValueError("theta and the scaling factor must be positive")
        self.inv_freq = None

    def frequencies(self):
        """Angle a position of each pair, float64 [rotary_dim / 2]."""
        exponent = torch.arange(0, self.rotary_dim, 2, dtype=torch.float64) / self.rotary_dim
        return self.theta ** -exponent / self.factor

    def prepare(self, device, dtype):
        if self.inv_freq is None or self.inv_freq.device != torch.device(device):
            self.inv_freq = self.frequencies().to(torch.float32).to(device).contiguous()


@register_position_encoding("rotary_half_angles")
class RotaryHalfAngles(RotaryInterleaved):
    """The same angles on the other pairing: element i of the first ``rotary_dim`` dims turns with element
    i + rotary_dim / 2.  Like RotaryInterleaved it keeps no table: the kernels that use it compute
    position * inv_freq[i] and its cosine and sine in 32-bit themselves."""
    layout = "half"


@register_position_encoding("rotary_yarn")
class RotaryYarn(RotaryInterleaved):
    """Either pairing (``layout``: "half", the default, or "interleaved") with frequencies stretched by parts (YaRN: Peng et al., "YaRN: Efficient Context Window
    Extension of Large Language Models").  With n(t) = rotary_dim ln(original / (2 pi t)) / (2 ln theta), the place of the
    pair that turns t times over ``original`` positions: pairs up to floor(n(fast)) keep their frequency, pairs from
    ceil(n(slow)) on have theirs divided by ``factor``, those between move from one to the other linearly.  Cosines
    and sines are multiplied by 0.1 ln(factor) + 1."""

    def __init__(self, rotary_dim: int, theta: float, factor: float, original: float, fast: float, slow: float,
                 layout: str = "half"):
        super().__init__(rotary_dim, theta)
        if layout not in ("half", "interleaved"):
            raise ValueError(f"layout {layout!r} (interleaved or half)")
        self.layout = layout
        self.stretch, self.original, self.fast, self.slow = float(factor), float(original), float(fast), float(slow)
        if not (self.stretch > 0 and self.original > 0 and self.fast > 0 and self.slow > 0) or self.theta == 1.0:
            raise ValueError("factor, original, fast and slow must be positive, and theta another number than 1")
        self.magnitude = 0.1 * math.log(self.stretch) + 1.0

    def frequencies(self):
        plain = super().frequencies()
        place = lambda turns: self.rotary_dim * math.log(self.original / (2 * math.pi * turns)) / (2 * math.log(self.theta))   # noqa: E731
        low = max(math.floor(place(self.fast)), 0)
        high = min(math.ceil(place(self.slow)), self.rotary_dim - 1)
        ramp = ((torch.arange(plain.shape[0], dtype=torch.float64) - low) / max(high - low, 0.001)).clamp(0, 1)
        return plain / self.stretch * ramp + plain * (1 - ramp)
