"""RMS norm with the residual add fused in front of it.

``y = x / sqrt(mean(x^2) + eps) * gamma`` (crates/burn-lm-llama/src/nn/transformer.rs:60-62,
vector at :278-297).  The sum of squares, the root and the scaling are float32; the add that
precedes the norm in a block (transformer.rs:248-255) is done here, on the float32 residual.
"""
from __future__ import annotations

import torch

from .base import Gated, Joining, Norm, TensorSpec


class RMSNorm(Norm):
    """params: width, eps, single (default False; True: the stored weight is one number for all lanes, a tensor without
    dimensions), offset (default 0; 1: the stored weight is the distance from one) and scale (default 1: a factor on the
    result, folded into the weight, such as a logit scale in the last norm).  names: weight."""
    graph_safe = True

    def tensor_specs(self):
        return {self.names["weight"]: TensorSpec(() if self.params.get("single") else (self.params["width"],))}

    def bind(self, tensors, rt):
        self.rt = rt
        self.gamma = tensors[self.names["weight"]]
        if self.params.get("single"):      # the kernels read a weight per lane: the one number, once for each
            self.gamma = self.gamma.reshape(1).expand(self.params["width"])
        offset, scale = float(self.params.get("offset", 0.0)), float(self.params.get("scale", 1.0))
        if offset != 0.0 or scale != 1.0:
            self.gamma = ((self.gamma.double() + offset) * scale).float()
        self.gamma = self.gamma.contiguous()
        self.gamma32 = self.gamma.float()
        self.eps = float(self.params["eps"])

    def step_bytes(self, rows):
        return self.gamma.numel() * self.gamma.element_size()

    def rms_constants(self):
        return self.gamma, self.eps

    def post(self, terms):
        """A sublayer's results with this norm behind their sum, for the next norm's add."""
        return Joining(terms, self.gamma32, self.eps)

    def add_norm(self, h, delta, rows=None, write_h=True):
        n = h.shape[0] if rows is None else rows.shape[0]
        out = torch.empty(n, h.shape[1], dtype=self.rt.dtype, device=h.device)
        if isinstance(delta, Joining):
            return join(self.rt, h, delta, out, gamma=self.gamma32, eps=self.eps, rows=rows, write_h=write_h)
        if isinstance(delta, Gated):
            return self.rt.ops.add_rmsnorm(h, delta.y, self.gamma, self.eps, out, rows=rows, write_h=write_h,
                                           gate=delta.z, gate_bias=delta.bias, mult=delta.mult)
        return self.rt.ops.add_rmsnorm(h, delta, self.gamma, self.eps, out, rows=rows, write_h=write_h)


def join(rt, h, delta, out, gamma=None, eps=0.0, rows=None, write_h=True):
    """The kernel of a Joining: it joins h, and out (or None) takes the rows, normed with gamma and eps or as they are."""
    if any(t.row is not None for t in delta.terms):
        raise ValueError("results that are normed before they join the residual have no factor per token")
    return rt.ops.post_norm(h, [(t.y, t.scale, t.gamma, t.eps, t.bias) for t in delta.terms],
                            post=None if delta.gamma is None else (delta.gamma, delta.eps), fresh=delta.fresh, vec=delta.vec,
                            write_h=write_h, gamma=gamma, eps=eps, out=out, rows=rows)
