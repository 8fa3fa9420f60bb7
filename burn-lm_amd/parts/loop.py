"""What stands in front of each pass of layers that run several times with the same weights.

Ahead of pass ``t``: ``x <- W [x; x0] + step_t`` with ``x0`` the embedding's output and one stored vector per pass.  The
rows ``[x; x0]`` are one buffer per step: the embedding leaves its half in it once, every entry writes the other half (the
pending delta joined on the way).  The product's result is the residual's new start: it is handed on in float32, and the
next norm sums its partial planes and adds the vector."""
from __future__ import annotations

import torch

from .base import Gated, Joining, Part, TensorSpec, Term
from .norm_rms import join


class LoopEntry(Part):
    """params: width, times (number of passes).  names: proj [width, 2 width] (the residual's columns first), step
    [times, width]."""
    graph_safe = True

    def tensor_specs(self):
        d = self.params["width"]
        return {self.names["proj"]: TensorSpec((d, 2 * d)), self.names["step"]: TensorSpec((self.params["times"], d))}

    def bind(self, tensors, rt):
        self.rt = rt
        self.width = self.params["width"]
        self.w = rt.weight(tensors[self.names["proj"]])
        self.steps = [v.contiguous() for v in tensors[self.names["step"]].float()]

    def step_bytes(self, rows):
        return self.w.w.numel() * self.w.w.element_size() + 4 * self.width

    def step_flops(self, rows):
        return 2 * rows * self.w.w.numel()

    def begin(self, n_tokens, device):
        """The step's rows [x; x0]; the caller fills the second half with the embedding's output."""
        return torch.empty(n_tokens, 2 * self.width, dtype=self.rt.dtype, device=device)

    def enter(self, h, delta, both, t):
        """The residual h with its pending delta goes into the first half of the rows; what comes back starts it anew."""
        if isinstance(delta, Gated):
            raise ValueError("a loop's entry takes a plain delta or a Joining")
        if delta is not None and not isinstance(delta, Joining):
            delta = Joining([Term(delta)])
        x = both[:, :self.width]
        if delta is None:
            x.copy_(h)
        else:
            join(self.rt, h, delta, x, write_h=False)
        y = self.rt.linear(both, self.w, out_dtype=torch.float32, partials=True)
        return Joining([Term(y)], fresh=True, vec=self.steps[t])
