"""Time mixing: a matrix state with a decay per key channel and token, read before the token's own write with a bonus for it.

    h' = the row before (zeros for a request's first token); each s of r, k, v, g, w reads its own mix h + (h' - h) * mu_s
    r = W_r mix_r, k = W_k mix_k, v = W_v mix_v (heads x head_dim), gate = silu(W_g mix_g)
    w = exp(-exp(W_w2 tanh(W_w1 mix_w) + w0))   (heads x head_dim)
    per head, S [head_dim, head_dim] from zero:  o = (S + diag(u) k v^T)^T r;  S <- diag(w) S + k v^T
    out = W_o (concat_h(o_h / rms(o_h)) * norm * gate)

What a request carries between steps lies in its slot as one float32 vector: S of every head (as [heads, value, key]), then
the row it was fed last.  The mixes are formed in float32 by one kernel and rounded once; the two products of the decays
leave their sums in float32; tanh, exponentials, the bonus, the state, its sums and the norm of the outputs are float32.
"""

from __future__ import annotations

import torch

from ..weights.random import register_init_law
from ..weights.spec import BIAS, NORM, TensorSpec
from .base import Part, SlotState, register_part
from .linear import Linear

TOKEN_MIX = "token_mix"          # shares of the row before in a mix: uniform in [0, 1)
register_init_law(TOKEN_MIX, lambda shape, generator, device: torch.rand(shape, generator=generator, dtype=torch.float32, device=device))


class TimeMixing(Part):
    graph_safe = True
    MIXES = ("r", "k", "v", "g", "w")

    def __init__(self, spec, runtime):
        self.rt = runtime
        self.hidden = int(spec["hidden_size"])
        self.heads, self.dim, self.rank = int(spec["heads"]), int(spec["head_dim"]), int(spec["decay_rank"])
        self.eps = float(spec["eps"])
        self.name = spec.get("name", "mix")
        self.wide = self.heads * self.dim
        self.products = [Linear(runtime, self.hidden, [self.wide], [name]) for name in ("r", "k", "v", "g")]
        self.decay_down = Linear(runtime, self.hidden, [self.rank], ["w1"])
        self.decay_up = Linear(runtime, self.rank, [self.wide], ["w2"])
        self.out = Linear(runtime, self.wide, [self.hidden], ["o"])
        self.mu = self.decay_bias = self.bonus = self.norm_weight = None
        runtime.kernels.check_state_sizes(self.heads, self.dim, self.dim)
        self.state_size = self.wide * self.dim

    def _prefix(self, prefix):
        return f"{prefix}{self.name}."

    def _linears(self):
        return (*self.products, self.decay_down, self.decay_up, self.out)

    def _own_specs(self, p):
        return ([TensorSpec(f"{p}mu.{s}", (self.hidden,), TOKEN_MIX) for s in self.MIXES]
                + [TensorSpec(p + "w0", (self.wide,), BIAS), TensorSpec(p + "u", (self.heads, self.dim), BIAS),
                   TensorSpec(p + "norm", (self.wide,), NORM)])

    def tensors(self, prefix):
        p = self._prefix(prefix)
        return [spec for linear in self._linears() for spec in linear.tensors(p)] + self._own_specs(p)

    def load(self, fetch, prefix):
        p = self._prefix(prefix)
        for linear in self._linears():
            linear.load(fetch, p)
        *mu, w0, u, norm = (fetch(spec).to(torch.float32) for spec in self._own_specs(p))
        self.mu = torch.stack(mu).contiguous()
        self.decay_bias, self.bonus, self.norm_weight = w0.contiguous(), u.reshape(-1).contiguous(), norm.contiguous()

    def weight_bytes(self):
        return sum(linear.weight_bytes() for linear in self._linears())

    def cache_request(self):
        return SlotState((self.state_size + self.hidden,), torch.float32)

    def forward(self, x, ctx, cache, writes_cache: bool = True):
        k, dtype = self.rt.kernels, self.rt.dtype
        tokens = x.shape[0]
        mixes = ctx.arena.take((len(self.MIXES), tokens, self.hidden), dtype)
        k.token_shift(x, self.mu, cache.state, self.state_size, ctx, mixes)
        rkvg = ctx.arena.take((4, tokens, self.wide), dtype)
        for index, product in enumerate(self.products):
            product.forward(mixes[index], rkvg[index])
        down = ctx.arena.take((tokens, self.rank), torch.float32)
        self.decay_down.forward(mixes[4], down)
        low = ctx.arena.take((tokens, self.rank), dtype)
        k.tanh_rows(down, low)
        decay_logits = ctx.arena.take((tokens, self.wide), torch.float32)
        self.decay_up.forward(low, decay_logits)
        gated = ctx.arena.take((tokens, self.wide), dtype)
        k.time_mixing(rkvg, decay_logits, self.decay_bias, self.bonus, self.norm_weight, self.eps, x, self.heads, self.dim,
                      cache.state, self.state_size, ctx, gated)
        return self.out.forward(gated, ctx.arena.take((tokens, self.hidden), dtype))


register_part("mixer", "time_mixing", TimeMixing)
