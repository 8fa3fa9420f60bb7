"""Dense feed-forward with a squared ReLU: ``W_down max(W_up x, 0)^2`` without biases; the square is float32."""
from __future__ import annotations

from .base import FeedForward, TensorSpec


class DenseRelu2(FeedForward):
    """params: width, inner.  names: up, down."""
    graph_safe = True

    def tensor_specs(self):
        d, i = self.params["width"], self.params["inner"]
        return {self.names["up"]: TensorSpec((i, d)), self.names["down"]: TensorSpec((d, i))}

    def bind(self, tensors, rt):
        self.rt = rt
        self.w_up = rt.weight(tensors[self.names["up"]])
        self.w_down = rt.weight(tensors[self.names["down"]])

    def step_bytes(self, rows):
        return sum(w.w.numel() * w.w.element_size() for w in (self.w_up, self.w_down))

    def step_flops(self, rows):
        return 2 * rows * (self.w_up.w.numel() + self.w_down.w.numel())

    def forward(self, x, step):
        rt = self.rt
        z = rt.linear(x, self.w_up)
        return rt.linear(rt.ops.relu2(z, z), self.w_down, partials=True)     # in place
