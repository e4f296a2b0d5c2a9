"""Two mixers that read the same input, joined by fixed factors: y = left_scale * left(h) + right_scale * right(h).
Each side keeps its own cache or state (CombinedCache members ``left`` and ``right``).

Both sides offer ``w_in``, ``w_o``, ``branch_width`` and ``branch_into``: the two input matrices are stacked, so that one
product serves both, and so are the output matrices, side by side: each side writes what its output matrix reads, times its
factor (in 32-bit, before it is rounded), into its columns of one tensor, and one product adds the two."""
from __future__ import annotations

from .base import CombinedCache, Mixer, register_mixer


@register_mixer("scaled_pair")
class ScaledPair(Mixer):
    lazy_input = True

    def __init__(self, width: int, left: Mixer, right: Mixer, left_scale: float = 1.0, right_scale: float = 1.0):
        self.width, self.left, self.right = int(width), left, right
        self.left_scale, self.right_scale = float(left_scale), float(right_scale)
        self.w_in = self.w_o = None

    def children(self):
        return [self.left, self.right]

    def cache_requirement(self):
        return CombinedCache([("left", self.left.cache_requirement()), ("right", self.right.cache_requirement())])

    def prepare(self, device, dtype):
        import torch
        if self.w_in is not None:
            return
        for side in (self.left, self.right):
            side.prepare(device, dtype)
        wl, wr = self.left.w_in, self.right.w_in
        if wl.dtype != wr.dtype or self.left.w_o.dtype != self.right.w_o.dtype:
            raise ValueError("the two sides' matrices are stored in different formats")
        self.w_in, self.right_base = torch.cat([wl, wr]).contiguous(), wl.shape[0]
        self.left.w_in, self.right.w_in = self.w_in[:self.right_base], self.w_in[self.right_base:]
        n = self.left.branch_width
        self.w_o = torch.cat([self.left.w_o, self.right.w_o], dim=1).contiguous()
        self.left.w_o, self.right.w_o = self.w_o[:, :n], self.w_o[:, n:]

    def forward(self, x, step, cache, add_to=None):
        import torch
        ops, n = self.ops, self.left.branch_width
        sums = ops.linear(x, self.w_in, out_dtype=torch.float32)
        joined = torch.empty((sums.shape[0], n + self.right.branch_width), dtype=ops.act_dtype, device=sums.device)
        self.left.branch_into(joined[:, :n], self.left_scale, sums, 0, step, cache.sub("left"))
        self.right.branch_into(joined[:, n:], self.right_scale, sums, self.right_base, step, cache.sub("right"))
        return ops.linear(joined, self.w_o, add_to=add_to)
