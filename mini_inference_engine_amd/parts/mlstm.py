"""Matrix memory with exponential gates (the mLSTM of Beck et al., "xLSTM: Extended Long Short-Term Memory").

q = W_q h * dim^(-1/2) and k = W_k h of ``dim`` numbers a head, v = W_v h of ``vdim``.  Per head a log input gate
i = cap tanh((W_i h + b_i) / cap) and a log forget gate f = logsigmoid(cap tanh((W_f h + b_f) / cap)).  Per head a memory
S [dim, vdim], a normaliser n [dim] and a running maximum m, all zero before a request's first token:
    m' = max(f + m, i);   S <- exp(f + m - m') S + exp(i - m') k v^T;   n likewise with k alone;   m <- m'
    o = S^T q / (max(|n . q|, exp(-m)) + 1e-6).
Each head's o is divided by its root mean square, the heads are concatenated, multiplied by a weight of all heads' size and
by sigmoid(W_g h), and go through the output projection.  Gates, maximum, memory, normaliser and norm are 32-bit; memory,
normaliser and maximum live in the request's state slot, so a portion that starts anywhere goes on from what it holds.

One product computes everything that reads h; one backend call does the rest.
"""
from __future__ import annotations

from dataclasses import dataclass

from .base import CacheRequirement, Mixer, ParamSpec, register_mixer

DEFAULT_NAMES = dict(q="q", k="k", v="v", g="g", i="i", i_bias="i.b", f="f", f_bias="f.b", norm="norm", o="o")


@dataclass(frozen=True)
class MatrixMemory(CacheRequirement):
    """Per request: the memory [heads, dim, vdim], its normaliser [heads, dim] and the running maximum [heads], float32."""
    heads: int
    dim: int
    vdim: int

    def allocate(self, num_pages, page_size, num_slots, device, act_dtype):
        import torch
        make = lambda *shape: torch.zeros((num_slots, *shape), dtype=torch.float32, device=device)       # noqa: E731
        return {"state": make(self.heads, self.dim, self.vdim), "normaliser": make(self.heads, self.dim), "maximum": make(self.heads)}

    def reset_slot(self, tensors, slot):
        for t in tensors.values():
            t[slot].zero_()


@register_mixer("mlstm")
class MatrixLSTM(Mixer):
    lazy_input = True

    def __init__(self, width: int, num_heads: int, dim: int, vdim: int, gate_cap: float, eps: float, prefix: str,
                 q_scale: float | None = None, tensor_names=None):
        self.width, self.num_heads, self.dim, self.vdim = int(width), int(num_heads), int(dim), int(vdim)
        self.gate_cap, self.eps, self.prefix = float(gate_cap), float(eps), prefix
        if not self.gate_cap > 0:
            raise ValueError(f"gate_cap {gate_cap} must be positive")
        self.q_scale = float(q_scale) if q_scale is not None else self.dim ** -0.5
        self.names = dict(DEFAULT_NAMES, **(tensor_names or {}))
        nk, nv = self.num_heads * self.dim, self.num_heads * self.vdim
        self.cols = dict(q=0, k=nk, v=2 * nk, g=2 * nk + nv, i=2 * nk + 2 * nv, f=2 * nk + 2 * nv + self.num_heads)

    def params(self):
        nm, w, H = self.names, self.width, self.num_heads
        nk, nv = H * self.dim, H * self.vdim
        name = lambda k: f"{self.prefix}.{nm[k]}"        # noqa: E731
        return [ParamSpec.stacked("w_in", [(name("q"), (nk, w)), (name("k"), (nk, w)), (name("v"), (nv, w)), (name("g"), (nv, w)),
                                           (name("i"), (H, w)), (name("f"), (H, w))]),
                ParamSpec.single("i_bias", name("i_bias"), (H,)),
                ParamSpec.single("f_bias", name("f_bias"), (H,)),
                ParamSpec.single("norm", name("norm"), (nv,), init="scale"),
                ParamSpec.single("w_o", name("o"), (w, nv))]

    def cache_requirement(self):
        return MatrixMemory(self.num_heads, self.dim, self.vdim)

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
        for attr in ("i_bias", "f_bias", "norm"):       # 32-bit whatever the checkpoint stores
            setattr(self, attr, getattr(self, attr).float().contiguous())

    @property
    def branch_width(self) -> int:
        return self.num_heads * self.vdim

    def branch_into(self, out, scale, sums, base, step, cache):
        """What the output matrix reads, times ``scale``, into ``out`` [T, branch_width] (None: a new tensor); ``sums``: the
        float32 sums of a product that holds this part's ``w_in`` rows from column ``base`` on."""
        cols = self.cols if base == 0 else {k: v + base for k, v in self.cols.items()}
        t = cache.tensors
        return self.ops.mlstm(sums, cols, self.num_heads, self.dim, self.vdim, self.i_bias, self.f_bias, self.gate_cap, self.q_scale,
                              self.norm, self.eps, t["state"], t["normaliser"], t["maximum"], step, out=out, scale=scale)

    def forward(self, x, step, cache, add_to=None, sums=None, base=0):
        import torch
        if sums is None:
            sums, base = self.ops.linear(x, self.w_in, out_dtype=torch.float32), 0
        return self.ops.linear(self.branch_into(None, 1.0, sums, base, step, cache), self.w_o, add_to=add_to)
