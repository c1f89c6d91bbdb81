"""RMSNorm (ampere_kv/runner.py:48-57): x * rsqrt(mean(x^2) + eps), rounded to the activation dtype, then
times the weight.  Statistics are formed in float32.  The weight is kept in float32 (a widening of what the
file stores, so the product equals the reference's).

With `single_rounding` the norm is float32 from the statistics to the product with the weight, and a result is
rounded once, when it is stored (designs that say their norms are computed in 32-bit).  Such a norm takes no part in
the folding of norms into products; it can be added to the residual sum as it is computed (`add_normed`) and chained
with the norm that follows (`after`): the norm kernel of blocks that norm a branch before and after.

With `unit_offset` the file stores the weight around zero and the norm multiplies by 1 + w; the sum is formed once, at
load, in float32.  With `output_scale` the normed rows are multiplied by a constant as well (a model whose logits are
its head's product times a constant puts it on its final norm): the weight takes it once, at load, in float32.

With `scalar` the norm has ONE weight for all coordinates, stored as a tensor without axes; the vector the kernels read is
filled with it once, at load."""

from __future__ import annotations

import torch

from ..weights.random import NORM_STD, _normal, register_init_law
from ..weights.spec import NORM, TensorSpec
from .base import Norm, NormedDelta, NormedPair, ScaledDelta, StreamSums, UnnormedRows, register_part  # noqa: F401  (StreamSums is found here too)


NORM_OFFSET = "norm_offset"          # a norm weight that is stored around zero and applied as 1 + w
register_init_law(NORM_OFFSET, _normal(0.0, NORM_STD))


class RMSNorm(Norm):
    def __init__(self, spec, runtime):
        self.size = int(spec["size"])
        self.eps = float(spec["eps"])
        self.single_rounding = bool(spec.get("single_rounding", False))
        self.unit_offset = bool(spec.get("unit_offset", False))
        self.output_scale = float(spec.get("output_scale", 1.0))
        self.scalar = bool(spec.get("scalar", False))
        self.rt = runtime
        self.weight: torch.Tensor | None = None

    @property
    def role(self) -> str:
        return NORM_OFFSET if self.unit_offset else NORM

    def tensors(self, name: str):
        return [TensorSpec(name, () if self.scalar else (self.size,), self.role)]

    def load(self, fetch, name: str):
        self.weight = fetch(self.tensors(name)[0]).to(torch.float32)
        self.weight = self.weight.expand(self.size).contiguous() if self.scalar else self.weight.contiguous()
        if self.unit_offset:
            self.weight += 1.0
        if self.output_scale != 1.0:
            self.weight *= self.output_scale

    def weight_bytes(self):
        return self.size * 4

    def forward(self, x: torch.Tensor, out: torch.Tensor) -> torch.Tensor:
        """x [..., size] in the activation dtype -> out of the same shape."""
        if self.single_rounding:
            raise NotImplementedError("a norm with one rounding reads the float32 residual sum (forward_residual, after)")
        self.rt.kernels.rmsnorm(x.view(-1, self.size), self.weight, self.eps, out.view(-1, self.size))
        return out

    def forward_residual(self, stream: torch.Tensor, delta: torch.Tensor | None, out: torch.Tensor,
                         delta_scale: float = 1.0) -> torch.Tensor:
        """stream [tokens, size] float32 is the residual sum; `delta` (activation dtype), times `delta_scale`, is added
        to it in float32 first, then the sum is normed into `out` (activation dtype)."""
        if self.single_rounding:
            self.rt.kernels.norm_add_norm(stream, delta, None, 0.0, self.weight, self.eps, out, delta_scale=delta_scale)
            return out
        if delta_scale != 1.0:
            raise NotImplementedError("only a norm with one rounding adds a branch times a constant")
        self.rt.kernels.add_rmsnorm(stream, delta, self.weight, self.eps, out)
        return out

    def add_normed(self, stream: torch.Tensor, delta: torch.Tensor) -> None:
        if not self.single_rounding:
            raise NotImplementedError("only a norm with one rounding is added to the residual sum as it is computed")
        self.rt.kernels.norm_add_norm(stream, delta, self.weight, self.eps, None, 0.0, None)

    def after(self, stream, pending, out):
        if isinstance(pending, NormedPair) and self.single_rounding:       # one kernel: norm both branches, add, norm
            self.rt.kernels.norm_add_norm(stream, pending.delta, pending.weight, pending.eps, self.weight, self.eps, out,
                                          delta_scale=pending.scale, delta2=pending.second, post_weight2=pending.second_weight)
            return out
        if isinstance(pending, ScaledDelta) and self.single_rounding:      # one kernel: add the branch times its constant, norm
            self.rt.kernels.norm_add_norm(stream, pending.delta, None, 0.0, self.weight, self.eps, out,
                                          delta_scale=pending.scale, **pending.extras())
            return out
        if (pending is None or not isinstance(pending, NormedDelta)
                or not (self.single_rounding and type(pending.norm) is RMSNorm and pending.norm.single_rounding)):
            return super().after(stream, pending, out)
        self.rt.kernels.norm_add_norm(stream, pending.delta, pending.norm.weight, pending.norm.eps, self.weight, self.eps, out)
        return out

    def pending(self, stream: torch.Tensor, delta: torch.Tensor | None, stream_out: torch.Tensor, arena) -> "PendingNorm":
        """`forward_residual` not yet computed: for a consumer whose first product can compute it itself."""
        if self.single_rounding:
            return None
        return PendingNorm(self, stream, delta, stream_out, arena)

    def fold_gain(self):
        return None if self.single_rounding else self.weight

    def scaled(self, stream: torch.Tensor, sums: "StreamSums", arena) -> "ScaledNorm":
        """The norm of a residual sum whose rows' sums of squares are already known (`StreamSums`): for a consumer
        whose first product can norm its rows itself from them."""
        if self.single_rounding:
            return None
        return ScaledNorm(self, stream, sums, arena)


class ScaledNorm(UnnormedRows):
    """norm(stream) for a stream whose sums of squares are at hand, before anybody has computed it.  Like
    `PendingNorm` it is read exactly once, through a `Linear` or the gated product: where the kernel set's product
    norms its rows itself (`linear_scaled`) it does; otherwise the rows are normed by the norm's own kernel."""

    moved = False               # the residual sum stays where it is

    def __init__(self, norm: RMSNorm, stream, sums: StreamSums, arena):
        self.norm, self.stream, self.sums, self.arena = norm, stream, sums, arena
        self.shape = (stream.shape[0], norm.size)
        self.dtype = norm.rt.dtype
        self._used = False

    def _once(self):
        if self._used:
            raise RuntimeError("rows that were handed on unnormed can be read once")
        self._used = True

    def product(self, weight, out: torch.Tensor, bias: torch.Tensor | None = None) -> bool:
        kernels = self.norm.rt.kernels
        if self.sums.rows is not None:      # a step of many rows: the rows times this norm's weight are at hand
            if self.sums.gain is not self.norm.weight or not kernels.scales_rows_in_product(self.shape[0], weight, out.dtype, self.sums):
                return False
            self._once()
            kernels.linear_rowscaled(self.sums.rows, self.sums.sums, self.norm.eps, weight, out, bias=bias)
            return True
        if not kernels.norms_rows_in_product(self.shape[0], weight, out.dtype):
            return False
        self._once()
        kernels.linear_scaled(self.stream, self.sums.sums, self.norm.weight, self.norm.eps, weight, out, bias=bias)
        return True

    def rows(self) -> torch.Tensor:
        self._once()
        out = self.arena.take(self.shape, self.dtype)
        return self.norm.forward_residual(self.stream, None, out)


class PendingNorm(UnnormedRows):
    """The rows norm(stream + delta) before anybody has computed them.  A part that `takes_pending_norm` reads them
    exactly once, through a `Linear` or the kernel set's gated product: where the kernel set's product can norm a few
    rows itself (`norm_in_product`), it does, and the new residual sum is then in `stream_out` (`moved` tells the
    block); otherwise the rows are normed here first, in place as `forward_residual` does."""

    def __init__(self, norm: RMSNorm, stream, delta, stream_out, arena):
        self.norm, self.stream, self.delta, self.stream_out, self.arena = norm, stream, delta, stream_out, arena
        self.shape = (stream.shape[0], norm.size)
        self.dtype = norm.rt.dtype
        self.moved = False          # the residual sum now lives in stream_out
        self._used = False

    def _once(self):
        if self._used:
            raise RuntimeError("rows that were handed on unnormed can be read once")
        self._used = True

    def product(self, weight, out: torch.Tensor, bias: torch.Tensor | None = None) -> bool:
        """out = these rows times `weight` (a packed matrix or a gated pair), plus `bias`, if the kernel set computes
        the norm inside that product; False if the caller has to ask for `rows()` and multiply itself."""
        kernels = self.norm.rt.kernels
        if not kernels.norm_in_product(self.shape[0], weight, out.dtype):
            return False
        self._once()
        kernels.linear_after_norm(self.stream, self.delta, self.norm.weight, self.norm.eps, self.stream_out, weight, out,
                                  bias=bias)
        self.moved = True
        return True

    def rows(self) -> torch.Tensor:
        """The rows, normed now by the norm's own kernel (the residual sum is updated in place)."""
        self._once()
        out = self.arena.take(self.shape, self.dtype)
        return self.norm.forward_residual(self.stream, self.delta, out)


register_part("norm", "rmsnorm", RMSNorm)
