"""What runs right before each pass of a looped stretch of layers: stream <- W [stream; embedding] + step_t, t the number of the
pass and ``embedding`` the stream as the embedding left it.

W is [width, 2 width]; the operand [stream | embedding] is one tensor of the step in the activation dtype (StepContext.shared),
whose right half the embedding fills and whose left half every pass writes anew.  The product's 32-bit sums are the new stream; the
step vector is added by whoever reads the stream next (kernels.api.BiasedBranch)."""
from __future__ import annotations

from ..kernels.api import BiasedBranch, Normed, NormedBranch, StreamCopy
from .base import ParamSpec, Part

SHARED = "stream_and_embedding"


class LoopEntry(Part):
    def __init__(self, width: int, times: int, weight_name: str, step_name: str):
        self.width, self.times = int(width), int(times)
        if self.times < 1:
            raise ValueError(f"{times} passes")
        self.weight_name, self.step_name = weight_name, step_name
        self.weight = self.steps = None

    def params(self):
        return [ParamSpec.single("weight", self.weight_name, (self.width, 2 * self.width)),
                ParamSpec.single("steps", self.step_name, (self.times, self.width))]

    def prepare(self, device, dtype):
        self.steps = self.steps.float().contiguous()

    def keep_embedding(self, step, width):
        """Where the embedding leaves its rows for this step's passes: [T, width] in the activation dtype."""
        import torch
        ids = step.input_ids
        joined = torch.empty((ids.shape[0], 2 * width), dtype=self.ops.act_dtype, device=ids.device)
        step.shared[SHARED] = joined
        return joined[:, width:]

    def forward(self, h, residual, step, turn):
        import torch
        joined = step.shared[SHARED]
        vector = None
        if isinstance(h, NormedBranch):
            h = h.resolve()
        if isinstance(h, Normed):           # the last product of the block before may still be to be added
            h, vector = h.pending, getattr(h, "pending_bias", None)
        elif isinstance(h, BiasedBranch):
            h, vector = h.value, h.bias
        elif isinstance(h, StreamCopy):
            h = None
        self.ops.stream_copy(h, residual, joined[:, :self.width], x_bias=vector)
        return BiasedBranch(None, self.steps[turn]), self.ops.linear(joined, self.weight, out_dtype=torch.float32)
