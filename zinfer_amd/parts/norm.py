from __future__ import annotations

from typing import Dict

import torch

from .. import ops
from ..config.specs import LayerNormSpec, RmsNormSpec
from .base import Norm, TensorDecl, register_part
from .linear import place_gain


class RmsNorm(Norm):
    """n = x * w / sqrt(mean(x^2) + eps) (`src/kernel/core/cpu.zig:38-48,73-110`); reads the
    float32 residual stream, writes the activation dtype.

    Under bfloat16 on the GPU the norm can be taken apart by the products around it: the
    weight-streaming product folds it in (``LazyRmsNorm.fold_into``), and the product that
    last adds into the residual can leave the norm's inputs or its whole result
    (``residual_sum``)."""
    graph_safe = True
    defers = True
    kernel_modules = ("elementwise",)


    def declare(self) -> Dict[str, TensorDecl]:
        return {self.prefix + self.spec.weight_name: TensorDecl((self.spec.width,), init="gain")}

    def bind(self, tensors) -> None:
        self.gain = place_gain(tensors[self.prefix + self.spec.weight_name], self.ctx)

    def forward(self, x: torch.Tensor, out: torch.Tensor) -> torch.Tensor:
        ops.rmsnorm(x, self.gain, float(self.spec.eps), out)
        return out

    def deferred(self, x: torch.Tensor, make_out, left=None):
        if not (x.is_cuda and self.ctx.compute_dtype == torch.bfloat16):
            return None
        given = left if left is not None and left.fits(self, x) else None
        return LazyRmsNorm(self, x, make_out, given)

    def residual_sum(self, linear, a: torch.Tensor, out: torch.Tensor, step) -> bool:
        if a.dtype != torch.bfloat16:
            return False
        M, N, K = a.shape[0], linear.out_features, linear.in_features
        if ops.norm_emit_plan(M, N, K, linear.weight, linear.tiled) is not None:
            xg = step.scratch("normed_by_gain", out.shape, torch.bfloat16)
            sq = step.scratch("normed_squares", (N // 16, 16), torch.float32)
            ops.gemm_emit(a, linear.weight, out, self.gain, xg, sq)
            step.norm_ready = GivenRmsNorm(self, out, xg, sq)
            return True
        if ops.sum_norm_plan(M, N, K, linear.weight, linear.tiled) is not None:
            normed = step.scratch("normed_by_sum", out.shape, torch.bfloat16)
            ops.gemm_sum_norm(a, linear.weight, out, self.gain, float(self.spec.eps), normed)
            step.norm_ready = DoneRmsNorm(self, out, normed)
            return True
        return False


class GivenRmsNorm:
    """What the kernel that last added into the residual rows ``x`` left for ``norm``:
    xg = bfloat16(x * gain) and sq [width / 16, 16], the sums of x^2 over each 16 columns per
    token (``ops.gemm_emit``)."""

    def __init__(self, norm: "RmsNorm", x: torch.Tensor, xg: torch.Tensor, sq: torch.Tensor):
        self.norm, self.x, self.xg, self.sq = norm, x, xg, sq

    def fits(self, norm, x: torch.Tensor) -> bool:
        return self.norm is norm and self.x.data_ptr() == x.data_ptr() and self.x.shape == x.shape


class DoneRmsNorm:
    """The norm of the residual rows ``x`` already run by the kernel that last added into them
    (``ops.gemm_sum_norm``): ``normed`` holds the result."""

    def __init__(self, norm: "RmsNorm", x: torch.Tensor, normed: torch.Tensor):
        self.norm, self.x, self.normed = norm, x, normed

    def fits(self, norm, x: torch.Tensor) -> bool:
        return self.norm is norm and self.x.data_ptr() == x.data_ptr() and self.x.shape == x.shape


class LazyRmsNorm:
    """A norm that has not run yet: the residual rows and the norm's parameters.  A consumer
    whose first matrix product can fold the norm in (``Linear.forward``) takes it apart;
    anyone else calls ``materialize()`` and gets the normed activations (computed once).
    ``given``: what the producer of the rows already left of the norm, if anything: its
    inputs (``GivenRmsNorm``) or its whole result (``DoneRmsNorm``)."""

    def __init__(self, norm: "RmsNorm", x: torch.Tensor, make_out, given: GivenRmsNorm = None):
        self.x, self.gain, self.eps = x, norm.gain, float(norm.spec.eps)
        self.shape = x.shape
        self._norm, self._make_out, self._out = norm, make_out, None
        if isinstance(given, DoneRmsNorm):
            given, self._out = None, given.normed
        self.given = given

    @property
    def done(self) -> bool:
        return self._out is not None

    def materialize(self) -> torch.Tensor:
        if self._out is None:
            self._out = self._make_out()
            self._norm.forward(self.x, self._out)
        return self._out

    def fold_into(self, linear, out: torch.Tensor, swiglu: bool = False) -> bool:
        """out = norm(x) W^T (with ``swiglu`` the activation of a stacked gate/up weight) in
        the weight-streaming product, from the residual rows or from what their producer
        left; False (and nothing done) where that kernel does not cover the sizes."""
        M, K = self.shape
        if self.done or not linear.tiled:
            return False
        if swiglu:
            if M > ops.NORM_FOLD_MAX_M:
                return False
        elif ops.norm_gemm_plan(M, linear.out_features, K, linear.weight, True) is None:
            return False
        if self.given is not None:
            ops.gemm_given(self.given.xg, self.given.sq, self.eps, linear.weight, out,
                           swiglu=swiglu)
        else:
            ops.norm_gemm(self.x, self.gain, self.eps, linear.weight, out, swiglu=swiglu)
        return True


class LayerNorm(Norm):
    """n = (x - mean) / sqrt(mean((x - mean)^2) + eps) * w + b, all in 32-bit; reads the float32
    residual stream (or a branch's float32 output), writes the activation dtype, or adds its
    result to a float32 destination (``forward_add``: a norm after a sublayer, ahead of the
    residual sum; the sublayer's output bias, if it leaves one, joins on the way in).  Not centred it is an RMS norm with a bias."""
    graph_safe = True
    adds_input_bias = True
    kernel_modules = ("norms",)

    def declare(self) -> Dict[str, TensorDecl]:
        s = self.spec
        d = {self.prefix + s.weight_name: TensorDecl(
            (s.width,), init="gain" if s.gain_offset == 0.0 else "normal")}
        if s.bias_name is not None:
            d[self.prefix + s.bias_name] = TensorDecl((s.width,))
        return d

    def bind(self, tensors) -> None:
        s = self.spec
        self.gain = place_gain(tensors[self.prefix + s.weight_name], self.ctx)
        if s.gain_offset != 0.0:
            # a weight stored around zero: the gain is the offset plus the weight, added once
            # in 32-bit
            self.gain = (self.gain + float(s.gain_offset)).contiguous()
        self.bias = place_gain(tensors[self.prefix + s.bias_name], self.ctx) \
            if s.bias_name is not None else None

    def forward(self, x: torch.Tensor, out: torch.Tensor) -> torch.Tensor:
        ops.norm_rows(x, self.gain, self.bias, float(self.spec.eps), out, bool(self.spec.centred))
        return out

    def forward_add(self, x: torch.Tensor, residual: torch.Tensor, x_bias=None) -> None:
        """residual += norm(x + x_bias), in 32-bit."""
        ops.norm_rows(x, self.gain, self.bias, float(self.spec.eps), residual,
                      bool(self.spec.centred), add=True, x_bias=x_bias)

    def forward_embedding(self, table: torch.Tensor, ids: torch.Tensor, scale: float,
                          x: torch.Tensor, then: "Norm" = None, out: torch.Tensor = None) -> bool:
        """x = norm(table[ids] * scale) in one kernel, and where ``then`` is a norm of this kind
        (neither centred nor with a bias) out = then(x) in the same; says whether it was."""
        fused = out is not None and isinstance(then, LayerNorm) and then.plain
        ops.embed_norm(table, ids, self.gain, float(self.spec.eps), x, scale,
                       then.gain if fused else None, float(then.spec.eps) if fused else 0.0,
                       out if fused else None)
        return fused

    @property
    def plain(self) -> bool:
        """An RMS norm with a gain and nothing else."""
        return not self.spec.centred and self.spec.bias_name is None

    def forward_add_store(self, x: torch.Tensor, residual: torch.Tensor,
                          out: torch.Tensor) -> bool:
        """residual += norm(x) and out = residual in ``out``'s type in one kernel (for a block
        whose next sublayer reads the stream as it is), if the width allows; False (and nothing
        done) otherwise."""
        if not residual.is_cuda or not ops.norm_add_norm_covers(residual.shape[1]):
            return False
        ops.norm_add_store(x, self.gain, self.bias, float(self.spec.eps),
                           bool(self.spec.centred), residual, out)
        return True

    def forward_add_then(self, x: torch.Tensor, residual: torch.Tensor, then: "Norm",
                         out: torch.Tensor, x_bias=None) -> bool:
        """residual += norm(x + x_bias) and out = then(residual) in one kernel, if ``then`` is a
        norm of this kind and the width allows; False (and nothing done) otherwise."""
        if not isinstance(then, LayerNorm) or not residual.is_cuda \
                or not ops.norm_add_norm_covers(residual.shape[1]):
            return False
        ops.norm_add_norm(x, self.gain, self.bias, float(self.spec.eps), bool(self.spec.centred),
                          residual, then.gain, then.bias, float(then.spec.eps),
                          bool(then.spec.centred), out, y_bias=x_bias)
        return True


register_part("norm", RmsNormSpec, RmsNorm)
register_part("norm", LayerNormSpec, LayerNorm)
