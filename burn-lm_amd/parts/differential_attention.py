"""Differential attention: two attention maps per head over the same values, the second subtracted from the first.

``q`` and ``k`` hold two maps of ``dim`` lanes per head, ``[map 1 | map 2]``, each RMS-normed on its own with a weight of
``dim`` lanes; ``a_x = softmax(q_x k_x^T scale) v``; ``o = a_1 - lambda a_2`` with one number
``lambda = exp(lq1 . lk1) - exp(lq2 . lk2) + diff`` per layer; ``o / sqrt(mean(o^2) + eps) * (1 - diff)`` over the head's value
lanes, then the output projection.

The cache holds one key row of ``2 dim`` lanes per key-value head and token, both maps side by side.  A query of map x is
laid out over ``2 dim`` lanes with zeros in the other map's half, so that its product with a key row is its own map's
score: to the attention kernels this is grouped-query attention of ``2 heads`` query heads with keys of ``2 dim`` lanes, and
keys and values are read once for both maps.  The kernels hand their float32 results on; difference, norm and factor are
one kernel, which rounds once."""
from __future__ import annotations

import math

import torch

from .base import TensorSpec
from .sink_attention import SinkAttention


class DifferentialAttention(SinkAttention):
    """params: those of SinkAttention without rotation, gate, temperature and head mixing; dim is the size of one map;
    qk_norm "heads"; diff (the constant part of lambda), norm_eps (also the results' norm).
    names: those of SinkAttention and lq1, lk1, lq2, lk2."""
    graph_safe = True

    def __init__(self, params, names):
        if params.get("qk_norm") != "heads" or params.get("gate") or params.get("talk") or params.get("sink") not in (None, False):
            raise ValueError("differential attention: queries and keys are normed per head; no gate, sink or head mixing")
        super().__init__(dict(params, dim=2 * params["dim"], talk=False, sink=False), names)
        self.map_dim = params["dim"]

    def norm_lanes(self):
        return self.map_dim, self.map_dim

    def tensor_specs(self):
        specs = super().tensor_specs()
        specs.update({self.names[r]: TensorSpec((self.map_dim,)) for r in ("lq1", "lk1", "lq2", "lk2")})
        return specs

    def bind(self, tensors, rt):
        super().bind(tensors, rt)
        self.att_heads, self.diff = 2 * self.H, float(self.params["diff"])
        a, b, c, d = (tensors[self.names[r]].double().cpu() for r in ("lq1", "lk1", "lq2", "lk2"))
        self.lam = math.exp(float((a * b).sum())) - math.exp(float((c * d).sum())) + self.diff

    def mixing_flops(self, past, new):
        """Two maps: scores of dim lanes and weighted values each."""
        keys = sum(min(past + t + 1, self.window) for t in range(new)) if self.window else new * past + new * (new + 1) // 2
        return 2 * 2 * self.H * (self.map_dim + self.dv) * keys

    def _normed(self, qkv, step, view):
        q = torch.empty(qkv.shape[0], self.att_heads * self.dk, dtype=qkv.dtype, device=qkv.device)
        return self.rt.ops.qkv_norm(qkv, self.bias_in, self.q_norm_w, self.k_norm_w, self.norm_eps, step, view.block_table(step),
                                    view.k, view.v, view.page_size, self.att_heads, 2 * self.G, self.map_dim, self.dv,
                                    growth=self.growth, q_out=q)

    def attend(self, q, step, view):
        maps = self._attend(q, step, view, dtype=torch.float32)
        out = torch.empty(q.shape[0], self.H * self.dv, dtype=self.rt.dtype, device=q.device)
        return self.rt.ops.map_difference(maps, out, step, self.H, self.dv, self.lam, self.norm_eps, 1.0 - self.diff)
