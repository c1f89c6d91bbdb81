"""A matrix memory with exponential gates per head, kept in range by a running maximum.

    q = W_q h * head_dim^(-1/2), k = W_k h (heads x head_dim), v = W_v h (heads x value_dim)
    per head: log input gate i = cap tanh((W_i h + b_i) / cap), log forget gate f = logsigmoid(cap tanh((W_f h + b_f) / cap))
    S [head_dim, value_dim], n [head_dim] and m from zero:
        m' = max(f + m, i);  S <- exp(f + m - m') S + exp(i - m') k v^T;  n <- exp(f + m - m') n + exp(i - m') k
        o = S^T q / (max(|n . q|, exp(-m')) + read_eps)
    out = W_o (concat_h(o_h / rms(o_h)) * norm * sigmoid(W_g h))

What a request carries between steps lies in its slot as one float32 vector: S and n of every head (as [heads, value_dim +
1, head_dim] - n is one more column of S, whose value is 1 for every token), then the heads' m.  All matrices that read h
are one product; gates, maxima, exponentials, the state, its sums and the norm of the outputs are float32.
"""

from __future__ import annotations

import torch

from ..weights.spec import BIAS, NORM, TensorSpec
from .base import Part, SlotState, register_part
from .linear import Linear


class MatrixMemory(Part):
    graph_safe = True

    def __init__(self, spec, runtime):
        self.rt = runtime
        self.hidden = int(spec["hidden_size"])
        self.heads, self.dim, self.vdim = int(spec["heads"]), int(spec["head_dim"]), int(spec["value_dim"])
        self.cap, self.read_eps, self.eps = float(spec["gate_cap"]), float(spec["read_eps"]), float(spec["eps"])
        self.name = spec.get("name", "mix")
        if self.cap <= 0:
            raise ValueError(f"the gates' cap is positive, got {self.cap}")
        self.qk, self.vs = self.heads * self.dim, self.heads * self.vdim
        self.into = Linear(runtime, self.hidden, [self.qk, self.qk, self.vs, self.vs, self.heads, self.heads],
                           ["q", "k", "v", "g", "i", "f"])
        self.out = Linear(runtime, self.vs, [self.hidden], ["o"])
        self.i_bias = self.f_bias = self.norm_weight = None
        runtime.kernels.check_state_sizes(self.heads, self.dim, self.vdim)
        self.top_at = self.heads * (self.vdim + 1) * self.dim
        # (a slot is a whole number of 16-byte pieces: its rows can then be read four floats at a time)
        self.state_size = (self.top_at + self.heads + 3) // 4 * 4

    def _prefix(self, prefix):
        return f"{prefix}{self.name}."

    def _own_specs(self, p):
        return [TensorSpec(p + "i.b", (self.heads,), BIAS), TensorSpec(p + "f.b", (self.heads,), BIAS),
                TensorSpec(p + "norm", (self.vs,), NORM)]

    def tensors(self, prefix):
        p = self._prefix(prefix)
        return self.into.tensors(p) + self.out.tensors(p) + self._own_specs(p)

    def load(self, fetch, prefix):
        p = self._prefix(prefix)
        self.into.load(fetch, p)
        self.out.load(fetch, p)
        self.i_bias, self.f_bias, self.norm_weight = (fetch(spec).to(torch.float32).contiguous() for spec in self._own_specs(p))

    def weight_bytes(self):
        return self.into.weight_bytes() + self.out.weight_bytes()

    def cache_request(self):
        return SlotState((self.state_size,), torch.float32)

    def forward(self, x, ctx, cache, writes_cache: bool = True):
        k, dtype = self.rt.kernels, self.rt.dtype
        tokens = x.shape[0]
        projected = ctx.arena.take((tokens, self.into.total_out), dtype)
        self.into.forward(x, projected)
        gated = ctx.arena.take((tokens, self.vs), dtype)
        k.matrix_memory(projected, self.i_bias, self.f_bias, self.cap, self.read_eps, self.norm_weight, self.eps, self.heads,
                        self.dim, self.vdim, cache.state, self.top_at, ctx, gated)
        return self.out.forward(gated, ctx.arena.take((tokens, self.hidden), dtype))


register_part("mixer", "matrix_memory", MatrixMemory)
