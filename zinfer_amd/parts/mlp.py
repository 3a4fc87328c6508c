from __future__ import annotations

from typing import Dict

import torch

from .. import ops
from ..config.specs import DenseMlpSpec, GatedMlpSpec, SwiGluSpec
from ..errors import ConfigError
from .base import FeedForward, TensorDecl, register_part
from .linear import Linear, place_gain, place_matrix


class SwiGluMlp(FeedForward):
    """d = W_down (silu(W_gate m) * W_up m), added to the residual
    (`src/model/runtime/optimized_decoder/layer.zig:194-201`, `src/kernel/core/cpu.zig:130-147`).
    gate and up rows are stacked into one matrix at load: each output keeps its own dot
    product."""
    graph_safe = True
    accepts_lazy_norm = True
    kernel_modules = ("elementwise", "gemm")


    def declare(self) -> Dict[str, TensorDecl]:
        s, p = self.spec, self.prefix
        return {p + s.gate_name: TensorDecl((s.intermediate_size, s.hidden_size)),
                p + s.up_name: TensorDecl((s.intermediate_size, s.hidden_size)),
                p + s.down_name: TensorDecl((s.hidden_size, s.intermediate_size))}

    def bind(self, tensors) -> None:
        s, p = self.spec, self.prefix
        g, u = tensors[p + s.gate_name], tensors[p + s.up_name]
        if g.dtype != u.dtype:
            g, u = g.float(), u.float()
        g, u = place_matrix(g, self.ctx), place_matrix(u, self.ctx)
        # bfloat16 on the GPU with sizes the MFMA kernels take: gate and up rows alternate in
        # groups of 16 and the activation runs in the product's epilogue
        self.fused = self.ctx.compute_dtype == torch.bfloat16 and g.shape[0] % 32 == 0 \
            and ops.can_fuse_swiglu(_probe(g))
        stacked = ops.interleave_gate_up(g, u) if self.fused else torch.cat([g, u], dim=0)
        del g, u
        self.gate_up = Linear(stacked)
        self.down = Linear(place_matrix(tensors[p + s.down_name], self.ctx))

    def forward(self, h, residual, step) -> None:
        T = h.shape[0]
        I = self.spec.intermediate_size
        act = self.ctx.act_dtype
        a = step.scratch("ff_act", (T, I), act)
        if hasattr(h, "materialize"):
            # a norm that has not run: the gate/up product folds it in where it can
            if self.fused and h.fold_into(self.gate_up, a, swiglu=True):
                self.down.forward(a, residual, accumulate=True, step=step)
                return
            h = h.materialize()
        if self.fused and h.dtype == torch.bfloat16:
            ops.gemm_swiglu(h, self.gate_up.weight, a, w_tiled=self.gate_up.tiled)
        else:
            gu = step.scratch("gate_up", (T, 2 * I), act)
            self.gate_up.forward(h, gu)
            ops.swiglu(gu, a)
        self.down.forward(a, residual, accumulate=True, step=step)


class _probe:
    """Shape and placement of the stacked gate/up matrix, without building it."""

    def __init__(self, g: torch.Tensor):
        self.is_cuda, self.dtype, self.shape = g.is_cuda, g.dtype, (2 * g.shape[0], g.shape[1])


class DenseMlp(FeedForward):
    """d = W_down act(W_up m), no gate, with biases if the specification says so; bias and
    activation (``ops.ACTIVATIONS``) run in 32-bit on the product's values."""
    graph_safe = True
    stores_output = True
    joins = True
    kernel_modules = ("elementwise", "gemm")

    def declare(self) -> Dict[str, TensorDecl]:
        s, p = self.spec, self.prefix
        d = {p + s.up_name: TensorDecl((s.intermediate_size, s.hidden_size)),
             p + s.down_name: TensorDecl((s.hidden_size, s.intermediate_size))}
        if s.bias:
            d[p + s.up_name + s.bias_suffix] = TensorDecl((s.intermediate_size,))
            d[p + s.down_name + s.bias_suffix] = TensorDecl((s.hidden_size,))
        return d

    def input_matrices(self, tensors):
        return [tensors[self.prefix + self.spec.up_name]]

    def output_matrix(self, tensors):
        s, p = self.spec, self.prefix
        return tensors[p + s.down_name], \
            tensors[p + s.down_name + s.bias_suffix] if s.bias else None

    def bind_joined(self, tensors) -> None:
        s, p = self.spec, self.prefix
        if s.activation not in ops.ACTIVATIONS:
            raise ConfigError(f"activation {s.activation!r}: known are {sorted(ops.ACTIVATIONS)}")
        self.up_bias = place_gain(tensors[p + s.up_name + s.bias_suffix], self.ctx) \
            if s.bias else None

    def bind(self, tensors) -> None:
        self.up = Linear(place_matrix(self.input_matrices(tensors)[0], self.ctx))
        down, bias = self.output_matrix(tensors)
        self.down = Linear(place_matrix(down, self.ctx))
        self.down_bias = place_gain(bias, self.ctx) if bias is not None else None
        self.bind_joined(tensors)

    def forward(self, h, residual, step, accumulate: bool = True) -> None:
        if hasattr(h, "materialize"):
            h = h.materialize()
        a = step.scratch("ff_act", (h.shape[0], self.spec.intermediate_size), self.ctx.act_dtype)
        self.up.forward(h, a)
        if self.up_bias is None:
            ops.activation(a, a, self.spec.activation)
        else:
            ops.bias_act_rows(a, self.up_bias, a, self.spec.activation)
        self.down.forward(a, residual, accumulate=accumulate,
                          step=step if accumulate and self.down_bias is None else None)
        if self.down_bias is not None:
            ops.add_row(residual, self.down_bias)

    def inner(self, rows, out, step, tail: int = 0, ones: int = 0) -> None:
        """Bias and activation from the input product's columns to what the output product reads;
        the last ``tail`` columns of ``out`` become ones and zeros (``ops.bias_act_rows``)."""
        ops.bias_act_rows(rows, self.up_bias, out, self.spec.activation, tail=tail, ones=ones)


class GatedMlp(FeedForward):
    """d = W_down (act(W_gate m) * W_up m) with any of ``ops.ACTIVATIONS`` and, if the
    specification says so, biases on all three.  gate and up rows are stacked into one matrix at
    load: each output keeps its own dot product.  Biases, activation and the product of the two
    run in 32-bit: for the tanh form of gelu in bfloat16, where the sizes allow, in the product's
    epilogue (gate and up rows then alternate in groups of 16), else on the product's rows.
    The output's bias may be left to a norm behind the part."""
    graph_safe = True
    stores_output = True
    leaves_bias = True
    kernel_modules = ("elementwise", "gemm")

    def __init__(self, spec: GatedMlpSpec, ctx, prefix):
        super().__init__(spec, ctx, prefix)
        if spec.activation not in ops.ACTIVATIONS:
            raise ConfigError(f"activation {spec.activation!r}: known are {sorted(ops.ACTIVATIONS)}")

    def declare(self) -> Dict[str, TensorDecl]:
        s, p = self.spec, self.prefix
        d = {p + s.gate_name: TensorDecl((s.intermediate_size, s.hidden_size)),
             p + s.up_name: TensorDecl((s.intermediate_size, s.hidden_size)),
             p + s.down_name: TensorDecl((s.hidden_size, s.intermediate_size))}
        if s.bias:
            for name, width in ((s.gate_name, s.intermediate_size),
                                (s.up_name, s.intermediate_size), (s.down_name, s.hidden_size)):
                d[p + name + s.bias_suffix] = TensorDecl((width,))
        return d

    def bind(self, tensors) -> None:
        s, p = self.spec, self.prefix
        g, u = tensors[p + s.gate_name], tensors[p + s.up_name]
        if g.dtype != u.dtype:
            g, u = g.float(), u.float()
        g, u = place_matrix(g, self.ctx), place_matrix(u, self.ctx)
        self.fused = s.activation == "gelu_tanh" and g.is_cuda and g.dtype == torch.bfloat16 \
            and self.ctx.compute_dtype == torch.bfloat16 \
            and ops.can_fuse_geglu(s.intermediate_size, s.hidden_size)
        self.gate_up = Linear(ops.interleave_gate_up(g, u) if self.fused
                              else torch.cat([g, u], dim=0))
        del g, u
        self.down = Linear(place_matrix(tensors[p + s.down_name], self.ctx))
        self.bias = self.down_bias = None
        if s.bias:
            both = [tensors[p + n + s.bias_suffix].to(torch.float32) for n in (s.gate_name, s.up_name)]
            self.bias = place_gain(ops.interleave_bias(*both) if self.fused else torch.cat(both),
                                   self.ctx)
            self.down_bias = place_gain(tensors[p + s.down_name + s.bias_suffix], self.ctx)

    def forward(self, h, residual, step, accumulate: bool = True, leave_bias: bool = False):
        T, I = h.shape[0], self.spec.intermediate_size
        act = self.ctx.act_dtype
        if hasattr(h, "materialize"):
            h = h.materialize()
        a = step.scratch("ff_act", (T, I), act)
        if self.fused:
            ops.gemm_geglu(h, self.gate_up.weight, self.bias, a)
        else:
            gu = step.scratch("gate_up", (T, 2 * I), act)
            self.gate_up.forward(h, gu)
            ops.gated_rows(gu, self.bias, a, self.spec.activation)
        last = self.down_bias is None
        self.down.forward(a, residual, accumulate=accumulate,
                          step=step if accumulate and last else None)
        if leave_bias:
            return self.down_bias
        if not last:
            ops.add_row(residual, self.down_bias)
        return None


register_part("feed_forward", SwiGluSpec, SwiGluMlp)
register_part("feed_forward", GatedMlpSpec, GatedMlp)
register_part("feed_forward", DenseMlpSpec, DenseMlp)
