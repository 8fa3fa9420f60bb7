"""Token embedding and output head.

``h = table[ids]`` with no scaling (crates/burn-lm-llama/src/nn/transformer.rs:95) into the
float32 residual stream; ``logits = x W_out^T`` without bias in float32 (transformer.rs:102).
A tied head uses the embedding table itself: the ``[vocab, width]`` table is the head's
``[d_out, d_in]`` matrix (the reference leaves tying as a TODO, transformer.rs:82-84)."""
from __future__ import annotations

import math

import torch

from .base import Joining, Part, TensorSpec, Term


class Embedding(Part):
    """params: vocab, width, copies (default 1; more: the residual starts as that many equal streams,
    [tokens, copies, width]), scale (default 1: every row is multiplied by it), position_base (default none; a number b: a
    sinusoidal vector of the token's position p is added, entry 2i the sine and entry 2i + 1 the cosine of
    p * b^(-2i/width); the angles are reduced in double precision), norm_eps (default none; a number: the looked-up rows
    pass an RMS norm with this eps before they are the residual, see normed), norm_offset (default 0; 1: that norm's stored
    weight is the distance from one).  names: weight, and norm where there is one."""
    graph_safe = True

    def tensor_specs(self):
        specs = {self.names["weight"]: TensorSpec((self.params["vocab"], self.params["width"]))}
        if self.params.get("norm_eps") is not None:
            specs[self.names["norm"]] = TensorSpec((self.params["width"],))
        return specs

    def bind(self, tensors, rt):
        self.rt = rt
        self.table = tensors[self.names["weight"]].contiguous()
        self.scale = float(self.params.get("scale", 1.0))
        base, d = self.params.get("position_base"), self.params["width"]
        self.turns = None      # full turns of entries 2i and 2i + 1 per position
        if base is not None:
            exponents = torch.arange((d + 1) // 2, dtype=torch.float64) * (-2.0 / d)
            self.turns = (float(base) ** exponents / (2.0 * math.pi)).to(rt.device)
        self.norm_w = None
        if self.params.get("norm_eps") is not None:
            self.norm_w = (tensors[self.names["norm"]].double() + float(self.params.get("norm_offset", 0.0))).float().contiguous()

    def normed(self, rows):
        """(residual, pending delta) for the first layer: without a norm the rows are the residual; with one the residual
        starts from the normed rows inside the kernel of the first layer's own norm."""
        if self.norm_w is None:
            return rows, None
        return torch.empty_like(rows), Joining([Term(rows, gamma=self.norm_w, eps=float(self.params["norm_eps"]))], fresh=True)

    @property
    def positional(self):
        return self.params.get("position_base") is not None

    def step_bytes(self, rows):
        return rows * self.params["width"] * self.table.element_size()      # the rows that are looked up

    def _rows(self, ids):
        copies = int(self.params.get("copies", 1))
        shape = (ids.shape[0], self.params["width"]) if copies == 1 else (ids.shape[0], copies, self.params["width"])
        return torch.empty(shape, dtype=torch.float32, device=ids.device)

    def forward_at(self, step, copy=None):
        """The rows of a step's tokens with their positions' vectors; copy (a view [tokens, width] in the activation
        dtype) receives them once more."""
        if int(self.params.get("copies", 1)) != 1 or self.scale != 1.0:
            raise ValueError("positions' vectors and copies of the embedding come with one unscaled stream")
        return self.rt.ops.embed_positions(self.table, step.token_ids, step.positions, self.turns, self._rows(step.token_ids),
                                           copy=copy, source=step.token_source)

    def forward(self, ids):
        if self.positional:
            raise ValueError("an embedding with positions' vectors needs the step: forward_at")
        h = self._rows(ids)
        return self.rt.ops.embed_gather(self.table, ids, h, self.scale)

    def forward_from(self, ids, source_rows, source_cell):
        """The same where some tokens are still on the device: row t is element source_rows[t] of the
        array whose address is in source_cell, where source_rows[t] >= 0.  An embedding without this
        method gets its tokens gathered by a separate launch before the step."""
        h = self._rows(ids)
        return self.rt.ops.embed_gather_from(self.table, ids, source_rows, source_cell, h, self.scale)


class LMHead(Part):
    """params: vocab, width, softcap (optional; a positive number c: logits <- c * tanh(logits / c)).
    names: weight (the embedding's name when tied)."""
    graph_safe = True

    def tensor_specs(self):
        return {self.names["weight"]: TensorSpec((self.params["vocab"], self.params["width"]))}

    def bind(self, tensors, rt):
        self.rt = rt
        self.weight = rt.weight(tensors[self.names["weight"]])
        self.softcap = float(self.params.get("softcap") or 0.0)

    def step_bytes(self, rows):
        return self.weight.w.numel() * self.weight.w.element_size() if rows else 0

    def step_flops(self, rows):
        return 2 * rows * self.weight.w.numel()

    def forward(self, x):
        logits = self.rt.linear(x, self.weight, out_dtype=torch.float32)
        return self.rt.ops.softcap(logits, self.softcap) if self.softcap > 0 else logits
