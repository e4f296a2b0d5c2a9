"""State space with one decay a head and step (Mamba-2: Dao and Gu, "Transformers are SSMs: Generalized Models and Efficient
Algorithms Through Structured State Space Duality").

One product of the input is laid out [z | x | B | C | dt]: z and x of ``heads * vdim`` numbers, B and C of ``groups * state``,
dt one a head.  x, B and C pass a causal convolution per channel with a bias and silu; dt <- softplus(dt + bias).  Head h
reads group h // (heads / groups) of B and C.  Per head a state S [state, vdim], zero before a request's first token:
    S <- exp(-exp(A_log) dt) S + dt B x^T,     y = S^T C + D x.
The heads' y times silu(z) is RMS-normed in ``norm_groups`` equal parts, each by its own root mean square, multiplied by a
weight and goes through the output projection.  Convolution, decays, steps, state and norm are 32-bit.  State and the
convolution's last inputs live in the request's state slot, which the cache zeroes when it hands the slot out, so a portion
that starts anywhere goes on from what the slot holds.
"""
from __future__ import annotations

from .base import CombinedCache, FixedState, Mixer, ParamSpec, register_mixer
from .input_conv import ConvTail

DEFAULT_NAMES = dict(w_in="in", conv="conv", conv_bias="conv.b", dt_bias="dt_bias", a_log="A_log", skip="D", norm="norm", o="o")


@register_mixer("state_space")
class StateSpace(Mixer):
    lazy_input = True

    def __init__(self, width: int, heads: int, vdim: int, state: int, groups: int, taps: int, norm_groups: int, eps: float,
                 prefix: str, tensor_names=None):
        self.width, self.num_heads, self.vdim, self.state_dim = int(width), int(heads), int(vdim), int(state)
        self.groups, self.taps, self.norm_groups = int(groups), int(taps), int(norm_groups)
        self.inner = self.num_heads * self.vdim
        if self.num_heads % self.groups:
            raise ValueError(f"{heads} heads do not split into {groups} groups")
        if self.inner % self.norm_groups:
            raise ValueError(f"{self.inner} numbers do not split into {norm_groups} equal parts")
        if self.taps < 1:
            raise ValueError("the convolution needs at least one tap")
        self.eps, self.prefix = float(eps), prefix
        self.names = dict(DEFAULT_NAMES, **(tensor_names or {}))
        gn = self.groups * self.state_dim
        self.channels = self.inner + 2 * gn
        self.z_col, self.conv_col, self.dt_col = 0, self.inner, self.inner + self.channels
        self.b_at, self.c_at = self.inner, self.inner + gn      # within the convolved columns

    def params(self):
        n, w, H = self.names, self.width, self.num_heads
        name = lambda k: f"{self.prefix}.{n[k]}"        # noqa: E731
        return [ParamSpec.single("w_in", name("w_in"), (self.inner + self.channels + H, w)),
                ParamSpec.single("conv", name("conv"), (self.channels, self.taps)),
                ParamSpec.single("conv_bias", name("conv_bias"), (self.channels,), init="zeros"),
                ParamSpec.single("dt_bias", name("dt_bias"), (H,)),
                ParamSpec.single("a_log", name("a_log"), (H,)),
                ParamSpec.single("skip", name("skip"), (H,), init="scale"),
                ParamSpec.single("norm", name("norm"), (self.inner,), init="scale"),
                ParamSpec.single("w_o", name("o"), (w, self.inner))]

    def cache_requirement(self):
        return CombinedCache([("memory", FixedState((self.num_heads, self.state_dim, self.vdim), "float32")),
                              ("conv", ConvTail(self.channels, self.taps))])

    def prepare(self, device, dtype):
        import torch
        if getattr(self, "_prepared", False):
            return
        self._prepared = True
        rows = self.w_in.shape[0]
        if rows % 16:       # the product kernels like whole tiles of weight rows: the sums get a few columns nobody reads
            padded = torch.zeros((-(-rows // 16) * 16, self.width), dtype=self.w_in.dtype, device=self.w_in.device)
            padded[:rows] = self.w_in
            self.w_in = padded
        for attr in ("conv", "conv_bias", "dt_bias", "a_log", "skip", "norm"):      # 32-bit whatever the checkpoint stores
            setattr(self, attr, getattr(self, attr).float().contiguous())
        self.rate = torch.exp(self.a_log)

    @property
    def branch_width(self) -> int:
        return self.inner

    def branch_into(self, out, scale, sums, base, step, cache):
        """What the output matrix reads, times ``scale``, into ``out`` [T, branch_width] (None: a new tensor); ``sums``: the
        float32 sums of a product that holds this part's ``w_in`` rows from column ``base`` on."""
        ops = self.ops
        u = ops.short_conv(sums, base + self.conv_col, self.channels, self.conv, self.conv_bias, cache.sub("conv").tensors["tail"],
                           step, activation="silu")
        return ops.state_space(u, self.b_at, self.c_at, sums, base + self.z_col, base + self.dt_col, self.num_heads, self.groups,
                               self.state_dim, self.vdim, self.dt_bias, self.rate, self.skip, self.norm_groups, self.norm, self.eps,
                               cache.sub("memory").state, step, out=out, scale=scale)

    def forward(self, x, step, cache, add_to=None, sums=None, base=0):
        import torch
        if sums is None:
            sums, base = self.ops.linear(x, self.w_in, out_dtype=torch.float32), 0
        return self.ops.linear(self.branch_into(None, 1.0, sums, base, step, cache), self.w_o, add_to=add_to)
