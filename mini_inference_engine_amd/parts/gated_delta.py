"""Gated delta rule with a decay per key channel.

Per head a state S [dim, vdim] (key channel i, value channel j), zero before a request's first token:
    S <- diag(g) S;   w = beta (v - S^T k);   S <- S + k w^T;   o = S^T q
q, k (``num_kv_heads`` heads of dim, each read by num_heads / num_kv_heads heads) and v (num_heads of vdim) are projections that
each pass a short causal convolution per channel (``conv`` taps) and silu; q and k are then unit vectors head by head
(x / sqrt(sum(x^2) + 1e-6)), q times ``q_scale`` (dim^(-1/2) unless given).  beta = sigmoid(W_b h) per head,
g = exp(-exp(A) softplus(W_a2 W_a1 h + dt_bias)) per head and key channel.  Each head's o is divided by its root mean square,
multiplied by a weight of vdim numbers (one for all heads) and by sigmoid(W_g2 W_g1 h), and goes through the output projection.
Decays, gates, unit vectors, state and the whole recurrence are 32-bit.  The state and the convolution's last inputs live in the
request's state slot, which the cache zeroes when it hands the slot out, so a portion that starts anywhere goes on from what the
slot holds.

One product computes everything that reads h; every stretch of its rows starts on a multiple of 16, and so do the inner sizes
of the two low-rank products (zero rows and columns between).
"""
from __future__ import annotations

from .base import CombinedCache, FixedState, Mixer, ParamSpec, register_mixer
from .input_conv import ConvTail

DEFAULT_NAMES = dict(q="q", k="k", v="v", q_conv="q.conv", k_conv="k.conv", v_conv="v.conv", beta="b", rate="A_log", a1="a1", a2="a2",
                     decay_bias="dt_bias", g1="g1", g2="g2", norm="norm", o="o")


def _up16(n: int) -> int:
    return -(-n // 16) * 16


@register_mixer("gated_delta")
class GatedDelta(Mixer):
    lazy_input = True

    def __init__(self, width: int, num_heads: int, num_kv_heads: int, dim: int, vdim: int, conv: int | None, decay_rank: int,
                 gate_rank: int, eps: float, prefix: str, q_scale: float | None = None, float32_output: bool = False, tensor_names=None):
        if num_heads % num_kv_heads:
            raise ValueError(f"{num_heads} heads are not a multiple of {num_kv_heads} query/key heads")
        self.width, self.num_heads, self.num_kv_heads = int(width), int(num_heads), int(num_kv_heads)
        self.dim, self.vdim = int(dim), int(vdim)
        if self.dim > 256 or self.vdim > 256:
            raise ValueError(f"states of {dim} x {vdim} a head are beyond the 256 x 256 the recurrence kernels take")
        self.conv = None if conv is None else int(conv)
        if self.conv is not None and self.conv < 1:
            raise ValueError("the convolution needs at least one tap")
        self.decay_rank, self.gate_rank = int(decay_rank), int(gate_rank)
        self.eps, self.prefix = float(eps), prefix
        self.q_scale = float(q_scale) if q_scale is not None else self.dim ** -0.5
        self.float32_output = bool(float32_output)
        self.names = dict(DEFAULT_NAMES, **(tensor_names or {}))
        nk, nv = self.num_kv_heads * self.dim, self.num_heads * self.vdim
        self.channels = 2 * nk + nv             # of the convolved projections, in the order of the columns
        self.k_at, self.v_at = nk, 2 * nk
        self.beta_col = _up16(self.channels)
        self.decay_col = self.beta_col + _up16(self.num_heads)
        self.gate_col = self.decay_col + _up16(self.decay_rank)
        self.columns = self.gate_col + _up16(self.gate_rank)

    def params(self):
        n, w, H = self.names, self.width, self.num_heads
        nk, nv = self.num_kv_heads * self.dim, H * self.vdim
        name = lambda k: f"{self.prefix}.{n[k]}"        # noqa: E731
        specs = [ParamSpec.stacked("w_in", [(name("q"), (nk, w)), (name("k"), (nk, w)), (name("v"), (nv, w)), (name("beta"), (H, w)),
                                            (name("a1"), (self.decay_rank, w)), (name("g1"), (self.gate_rank, w))]),
                 ParamSpec.single("rate", name("rate"), (H,)),
                 ParamSpec.single("w_decay", name("a2"), (H * self.dim, self.decay_rank)),
                 ParamSpec.single("decay_bias", name("decay_bias"), (H * self.dim,)),
                 ParamSpec.single("w_gate", name("g2"), (nv, self.gate_rank)),
                 ParamSpec.single("norm", name("norm"), (self.vdim,), init="scale"),
                 ParamSpec.single("w_o", name("o"), (w, nv))]
        if self.conv is not None:
            specs.append(ParamSpec.stacked("taps", [(name("q_conv"), (nk, self.conv)), (name("k_conv"), (nk, self.conv)),
                                                    (name("v_conv"), (nv, self.conv))]))
        return specs

    def cache_requirement(self):
        return CombinedCache([("memory", FixedState((self.num_heads, self.dim, self.vdim), "float32")),
                              ("conv", ConvTail(self.channels, self.conv or 1))])

    def prepare(self, device, dtype):
        import torch
        if getattr(self, "_prepared", False):
            return
        self._prepared = True
        spread, at = torch.zeros((self.columns, self.width), dtype=self.w_in.dtype, device=self.w_in.device), 0
        for col, n in ((0, self.channels), (self.beta_col, self.num_heads), (self.decay_col, self.decay_rank), (self.gate_col, self.gate_rank)):
            spread[col:col + n] = self.w_in[at:at + n]
            at += n
        self.w_in = spread
        for attr, rank in (("w_decay", self.decay_rank), ("w_gate", self.gate_rank)):
            w = getattr(self, attr)
            wide = torch.zeros((w.shape[0], _up16(rank)), dtype=torch.float32, device=w.device)
            wide[:, :rank] = w.float()
            setattr(self, attr, wide)
        if self.conv is None:
            self.taps = torch.ones((self.channels, 1), device=self.w_in.device)
        for attr in ("taps", "decay_bias", "norm"):         # 32-bit whatever the checkpoint stores
            setattr(self, attr, getattr(self, attr).float().contiguous())
        self.rate = torch.exp(self.rate.float())

    def forward(self, x, step, cache, add_to=None):
        import torch
        ops, nk = self.ops, self.k_at
        sums = ops.linear(x, self.w_in, out_dtype=torch.float32)
        u = ops.short_conv(sums, 0, self.channels, self.taps, None, cache.sub("conv").tensors["tail"], step, activation="silu")
        out = ops.gated_delta(u, 0, nk, 2 * nk, sums, self.beta_col, self.decay_col, self.gate_col, self.num_heads, self.num_kv_heads,
                              self.dim, self.vdim, self.w_decay, self.rate, self.decay_bias, self.w_gate, self.q_scale, self.norm,
                              self.eps, cache.sub("memory").state, step)
        if add_to is None and self.float32_output:
            return ops.linear(out, self.w_o, out_dtype=torch.float32)
        return ops.linear(out, self.w_o, add_to=add_to)
