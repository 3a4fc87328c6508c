from __future__ import annotations

from typing import Dict

import torch

from .. import ops
from ..config.specs import StateSpaceSpec
from ..errors import ConfigError
from .base import Mixer, StateNeed, StepHints, TensorDecl, register_part
from .linear import Linear, place_gain, place_matrix


class StateSpace(Mixer):
    """The mixer of ``StateSpaceSpec``.  z, x, B and C come from one product (the input matrix's
    rows without its last ones, filled up to the multiple of 64 the MFMA kernels' own order
    takes), the step sizes' numbers from a second one over those last rows that leaves its
    accumulators as 32-bit numbers (single tokens in bfloat16: the recurrence's kernel forms them
    itself, one launch less).  One kernel runs the short convolutions with bias and silu
    from the product's rows and the request's last rows; the recurrence's kernels form step size
    and decay a head and token and keep every request's matrices in its state slot (32-bit), the
    convolution's last rows behind them (32-bit); one more kernel applies the gate and norms the
    parts.  In bfloat16 long portions run in chunks side by side; which sequences do, and their
    chunks, is packed with the step's metadata (``step_hints``)."""
    graph_safe = True
    stores_output = True
    kernel_modules = ("gemm", "delta", "state_space", "recurrent")
    HINT_KEY = "state_space_chunks"
    ALIGN = 64

    def __init__(self, spec: StateSpaceSpec, ctx, prefix):
        super().__init__(spec, ctx, prefix)
        s = spec
        if min(s.n_heads, s.value_dim, s.state_dim, s.n_groups, s.conv_taps, s.norm_groups) < 1:
            raise ConfigError("InvalidDimensions: heads, sizes, groups and taps must be at least 1")
        if s.n_heads % s.n_groups != 0:
            raise ConfigError(f"InvalidGrouping: {s.n_heads} heads in {s.n_groups} groups")
        if s.n_heads * s.value_dim % s.norm_groups != 0:
            raise ConfigError(f"norm_groups={s.norm_groups} does not divide a row of "
                              f"{s.n_heads * s.value_dim}")
        if s.state_dim > ops.STATE_SPACE_MAX_STATE:
            raise ConfigError(f"state={s.state_dim}: the state-space kernels take up to "
                              f"{ops.STATE_SPACE_MAX_STATE} channels")
        if s.conv_taps > ops.SHORT_CONV_MAX_TAPS:
            raise ConfigError(f"conv={s.conv_taps}: the convolution kernel takes up to "
                              f"{ops.SHORT_CONV_MAX_TAPS} taps")
        self.inner = s.n_heads * s.value_dim
        self.bc_width = s.n_groups * s.state_dim
        self.conv_width = self.inner + 2 * self.bc_width
        # the matrices (whole 16 bytes), then the convolution's last rows
        self.matrix_size = ops.state_space_state_size(s.n_heads, s.state_dim, s.value_dim)
        self.state_size = (self.matrix_size + (s.conv_taps - 1) * self.conv_width + 3) // 4 * 4
        # only the bfloat16 kernels run in chunks
        if ctx.compute_dtype == torch.bfloat16:
            self.hint_key = self.HINT_KEY

    def declare(self) -> Dict[str, TensorDecl]:
        s, p = self.spec, self.prefix
        H = s.n_heads
        return {p + s.in_name: TensorDecl((self.inner + self.conv_width + H, s.hidden_size)),
                p + s.conv_name: TensorDecl((self.conv_width, s.conv_taps)),
                p + s.conv_bias_name: TensorDecl((self.conv_width,)),
                p + s.step_bias_name: TensorDecl((H,)),
                p + s.decay_log_name: TensorDecl((H,)),
                p + s.skip_name: TensorDecl((H,)),
                p + s.norm_name: TensorDecl((self.inner,), init="gain"),
                p + s.o_name: TensorDecl((s.hidden_size, self.inner))}

    def bind(self, tensors) -> None:
        s, p = self.spec, self.prefix
        w = tensors[p + s.in_name]
        rows = self.inner + self.conv_width
        wide = w[:rows]
        if rows % self.ALIGN:
            wide = torch.cat([wide, wide.new_zeros((-rows % self.ALIGN, wide.shape[1]))], dim=0)
        self.proj = Linear(place_matrix(wide.contiguous(), self.ctx))
        steps = place_matrix(w[rows:].contiguous(), self.ctx)
        self.step_proj = Linear(steps)
        # the rows as they lie, for the kernel that forms single tokens' step sizes itself
        self.step_rows = steps if steps.dtype == torch.bfloat16 and \
            self.ctx.compute_dtype == torch.bfloat16 and \
            ops.state_space_forms_steps(s.hidden_size) else None
        self.taps = place_gain(tensors[p + s.conv_name], self.ctx)
        self.conv_bias = place_gain(tensors[p + s.conv_bias_name], self.ctx)
        self.step_bias = place_gain(tensors[p + s.step_bias_name], self.ctx)
        self.decay_log = place_gain(tensors[p + s.decay_log_name], self.ctx)
        self.skip = place_gain(tensors[p + s.skip_name], self.ctx)
        self.gain = place_gain(tensors[p + s.norm_name], self.ctx)
        self.o = Linear(place_matrix(tensors[p + s.o_name], self.ctx))

    def cache_need(self):
        return StateNeed((self.state_size,), torch.float32)

    def step_hints(self, shape):
        lists = None if shape.fixed_shapes else ops.fixed_decay_chunk_lists(shape.q_lens)
        if lists is None:
            return None
        return StepHints(dict(zip(("chunks", "firsts", "shorts"), lists)))

    def forward(self, h, residual, step, cache, accumulate: bool = True) -> None:
        s = self.spec
        T = h.shape[0]
        act = self.ctx.act_dtype
        if hasattr(h, "materialize"):
            h = h.materialize()
        I, BC = self.inner, self.bc_width
        proj = step.scratch("space_proj", (T, self.proj.out_features), act)
        self.proj.forward(h, proj)
        single = step.max_q_len == 1
        if single and self.step_rows is not None:
            sizes = (h, self.step_rows)
        else:
            sizes = step.scratch("space_steps", (T, s.n_heads), torch.float32)
            self.step_proj.forward(h, sizes)
        xbc = step.scratch("space_xbc", (T, self.conv_width), act)
        ops.short_conv(proj[:, I:], self.taps, cache.state, self.matrix_size, step.state_slots,
                       step.seq_index, step.q_start, xbc, single_tokens=single,
                       bias=self.conv_bias)
        hints = step.hints.get(self.hint_key) if self.hint_key is not None else None
        lists = None
        if hints is not None and "chunks" in hints.arrays:
            lists = tuple(hints.arrays.get(n) for n in ("chunks", "firsts", "shorts"))
        y = step.scratch("space_out", (T, I), torch.float32)
        ops.state_space(xbc[:, :I], xbc[:, I:I + BC], xbc[:, I + BC:], sizes, self.decay_log,
                        self.step_bias, self.skip, cache.state, step.state_slots, step.q_start, y,
                        s.n_heads, s.n_groups, s.state_dim, s.value_dim, lists=lists,
                        single_tokens=single)
        mixed = step.scratch("space_mixed", (T, I), act)
        ops.gate_norm(y, self.gain, proj[:, :I], mixed, s.norm_groups, float(s.norm_eps))
        self.o.forward(mixed, residual, accumulate=accumulate, step=step if accumulate else None)


register_part("mixer", StateSpaceSpec, StateSpace)
