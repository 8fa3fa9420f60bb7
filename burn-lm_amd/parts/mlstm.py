"""Matrix memory with an exponential input gate (the mLSTM cell of xLSTM).

``q = W_q x * dim^-1/2``, ``k = W_k x`` (heads x dim), ``v = W_v x`` (heads x vdim); per head the logarithms of two gates,
``i = c tanh((W_i x + b_i) / c)`` and ``f = log sigmoid(c tanh((W_f x + b_f) / c))``; a matrix ``S``, a vector ``n`` and a
running maximum ``m``, all zero at a sequence's start:
``m_t = max(f + m_{t-1}, i)``, ``S_t = exp(f + m_{t-1} - m_t) S_{t-1} + exp(i - m_t) k v^T``, ``n_t`` likewise with ``k``,
``o = S_t^T q / (max(|n_t . q|, exp(-m_t)) + 1e-6)``.  Every head's ``o`` is divided by its root mean square, the heads are
concatenated, multiplied by a weight per lane and by ``sigmoid(W_g x)``, and projected.  State, gates, recurrence and norm
are float32 in every mode; so are the gates' logits, and in steps of few tokens the whole projection.  Such steps run in
one kernel that streams the state; prompts run in chunks of 64 tokens as float32 matrix products
(csrc/matrix_memory.hip)."""
from __future__ import annotations

import torch

from .base import Mixer, StateNeed, TensorSpec


class MLSTM(Mixer):
    """params: width, heads, dim, vdim, gate_cap, eps.  names: q, k, v, g, i, i_bias, f, f_bias, norm, o."""
    graph_safe = True
    CHUNKS_FROM = 8      # a step whose longest sequence brings at least this many tokens runs in chunks

    def tensor_specs(self):
        p, n = self.params, self.names
        d, H, dk, dv = p["width"], p["heads"], p["dim"], p["vdim"]
        return {n["q"]: TensorSpec((H * dk, d)), n["k"]: TensorSpec((H * dk, d)), n["v"]: TensorSpec((H * dv, d)),
                n["g"]: TensorSpec((H * dv, d)), n["i"]: TensorSpec((H, d)), n["i_bias"]: TensorSpec((H,)),
                n["f"]: TensorSpec((H, d)), n["f_bias"]: TensorSpec((H,)), n["norm"]: TensorSpec((H * dv,)),
                n["o"]: TensorSpec((d, H * dv))}

    def cache_need(self):
        p = self.params
        H, dk, dv = p["heads"], p["dim"], p["vdim"]
        return StateNeed((H, dk, dv), torch.float32), StateNeed((H, dk), torch.float32), StateNeed((H,), torch.float32)

    def bind(self, tensors, rt):
        self.rt = rt
        p, n = self.params, self.names
        self.H, self.dk, self.dv = p["heads"], p["dim"], p["vdim"]
        self.cap, self.eps, self.q_scale = float(p["gate_cap"]), float(p["eps"]), float(self.dk) ** -0.5
        ws = [tensors[n[r]] for r in ("q", "k", "v", "g")]
        # the gates' rows start at a multiple of eight, and all rows are one: a row range of it is a matrix of its own
        pad = lambda rows: [torch.zeros(-rows % 8, ws[0].shape[1], dtype=ws[0].dtype, device=ws[0].device)]
        ws += pad(sum(w.shape[0] for w in ws))
        self.gates_at = sum(w.shape[0] for w in ws)
        ws += [tensors[n["i"]], tensors[n["f"]]]
        ws += pad(sum(w.shape[0] for w in ws))
        if len({w.dtype for w in ws}) != 1:
            ws = [w.float() for w in ws]
        self.w_in = rt.weight(torch.cat(ws, dim=0))
        self.w_rows, self.w_gates = rt.weight(self.w_in.w[:self.gates_at]), rt.weight(self.w_in.w[self.gates_at:])
        self.w_o = rt.weight(tensors[n["o"]])
        self.bias_i, self.bias_f = (tensors[n[r]].float().contiguous() for r in ("i_bias", "f_bias"))
        self.norm_w = tensors[n["norm"]].float().contiguous()
        rt.ops.matrix_memory_init(rt.device)     # the kernels' shared memory, before any step is recorded
        self.in_chunks = rt.ops.matrix_memory_chunks_supported(self.dk, self.dv, rt.dtype)

    def step_bytes(self, rows):
        return sum(w.w.numel() * w.w.element_size() for w in (self.w_in, self.w_o))

    def step_flops(self, rows):
        return 2 * rows * (self.w_in.w.numel() + self.w_o.w.numel())

    def mixing_flops(self, past, new):
        return 5 * self.H * self.dk * (self.dv + 1) * new

    def forward(self, x, step, view):
        return self.output(self.scan(self.project(x, step), step, view))

    def project(self, x, step):
        """(rows [q | k | v | g], gate logits float32, whether the step runs in chunks)."""
        rt = self.rt
        if self.in_chunks and step.max_new >= self.CHUNKS_FROM and x.shape[0] > 4 * step.n_seqs:
            return rt.linear(x, self.w_rows), rt.linear(x, self.w_gates, out_dtype=torch.float32), True
        both = rt.linear(x, self.w_in, out_dtype=torch.float32)
        return both, both[:, self.gates_at:], False

    def scan(self, projected, step, view):
        """The recurrence over the step's tokens, each sequence from its own state -> [tokens, heads * vdim]."""
        proj, logits, chunks = projected
        out = torch.empty(proj.shape[0], self.H * self.dv, dtype=self.rt.dtype, device=proj.device)
        return self.rt.ops.matrix_memory(proj, logits, self.bias_i, self.bias_f, self.cap, self.q_scale, self.norm_w, self.eps,
                                         tuple(v.tensor for v in view), out, step, self.H, self.dk, self.dv, chunks)

    def output(self, mixed):
        return self.rt.linear(mixed, self.w_o, partials=True)
