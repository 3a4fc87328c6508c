from __future__ import annotations

import math
from typing import Dict

import torch

from .. import ops
from ..config.specs import FixedDecayAttentionSpec
from ..errors import ConfigError
from .base import Mixer, StateNeed, StepHints, TensorDecl, register_part
from .linear import Linear, place_gain, place_matrix


class FixedDecayAttention(Mixer):
    """The mixer of ``FixedDecayAttentionSpec``: q, k, v and the output gate come from one product
    over the stacked matrices; the recurrence's kernels take those rows as they are (silu, the
    rotation from a table made once a step and rotation, k's factor and the decay are theirs) and
    keep every request's matrices in its state slot (32-bit); one more kernel norms each head or
    the whole row and applies gain and gate.  In bfloat16 long portions run in chunks side by
    side; which sequences do, and their chunks, is packed with the step's metadata
    (``step_hints``)."""
    graph_safe = True
    stores_output = True
    joins = True
    kernel_modules = ("gemm", "fixed_decay", "recurrent")
    HINT_KEY = "fixed_decay_chunks"

    def __init__(self, spec: FixedDecayAttentionSpec, ctx, prefix):
        super().__init__(spec, ctx, prefix)
        s = spec
        if min(s.n_heads, s.head_dim, s.value_dim) < 1:
            raise ConfigError("InvalidDimensions: heads and head sizes must be at least 1")
        if s.head_dim > ops.FIXED_DECAY_MAX_KEY_DIM:
            raise ConfigError(f"InvalidHeadDim: dim={s.head_dim}: the recurrence's kernels take key "
                              f"sizes up to {ops.FIXED_DECAY_MAX_KEY_DIM}")
        if len(s.decay) != s.n_heads or any(not 0.0 <= float(g) <= 1.0 for g in s.decay):
            raise ConfigError(f"decay: {s.n_heads} numbers between 0 and 1, one a head, not "
                              f"{list(s.decay)}")
        if s.norm not in ("head", "row") or s.gate not in ops.GATE_KINDS:
            raise ConfigError(f"norm={s.norm!r} ('head' or 'row'), gate={s.gate!r} "
                              f"({sorted(ops.GATE_KINDS)})")
        if s.rotary is not None and (s.rotary.interleaved or not (
                0 < s.rotary.dims <= s.head_dim and s.rotary.dims % 2 == 0
                and len(s.rotary.frequencies) == s.rotary.dims // 2)):
            raise ConfigError(f"a rotation of {s.rotary.dims} elements in half-split pairs does "
                              f"not fit heads of {s.head_dim}")
        self.qk_width = s.n_heads * s.head_dim
        self.v_width = s.n_heads * s.value_dim
        self.state_size = ops.fixed_decay_state_size(s.n_heads, s.head_dim, s.value_dim)
        # only the bfloat16 kernels run in chunks
        if ctx.compute_dtype == torch.bfloat16:
            self.hint_key = self.HINT_KEY

    def declare(self) -> Dict[str, TensorDecl]:
        s, p = self.spec, self.prefix
        d = {p + s.q_name: TensorDecl((self.qk_width, s.hidden_size)),
             p + s.k_name: TensorDecl((self.qk_width, s.hidden_size)),
             p + s.v_name: TensorDecl((self.v_width, s.hidden_size)),
             p + s.gate_name: TensorDecl((self.v_width, s.hidden_size)),
             p + s.o_name: TensorDecl((s.hidden_size, self.v_width))}
        if s.norm_name is not None:
            d[p + s.norm_name] = TensorDecl((self.v_width,), init="gain")
        return d

    def input_matrices(self, tensors):
        s, p = self.spec, self.prefix
        return [tensors[p + n] for n in (s.q_name, s.k_name, s.v_name, s.gate_name)]

    def output_matrix(self, tensors):
        return tensors[self.prefix + self.spec.o_name], None

    def bind(self, tensors) -> None:
        rows = self.input_matrices(tensors)
        if len({t.dtype for t in rows}) > 1:
            rows = [t.float() for t in rows]
        self.proj = Linear(place_matrix(torch.cat(rows, dim=0), self.ctx))
        self.o = Linear(place_matrix(self.output_matrix(tensors)[0], self.ctx))
        self.bind_joined(tensors)

    def bind_joined(self, tensors) -> None:
        s, p = self.spec, self.prefix
        self.gain = place_gain(tensors[p + s.norm_name], self.ctx) \
            if s.norm_name is not None else None
        g = torch.tensor(s.decay, dtype=torch.float64)
        # (a decay of 0 forgets everything: 2^(-1e30 n) is 0 for n > 0 and 1 for n = 0)
        log2g = torch.tensor([math.log2(x) if x > 0.0 else -1e30 for x in g.tolist()],
                             dtype=torch.float64)
        self.decay = torch.stack([g, log2g]).to(torch.float32).to(self.ctx.device).contiguous()
        self.freq = None
        if s.rotary is not None:
            self.freq = torch.tensor(s.rotary.frequencies, dtype=torch.float64) \
                .to(torch.float32).to(self.ctx.device)

    def cache_need(self):
        return StateNeed((self.state_size,), torch.float32)

    def step_hints(self, shape):
        lists = None if shape.fixed_shapes else ops.fixed_decay_chunk_lists(shape.q_lens)
        if lists is None:
            return None
        return StepHints(dict(zip(("chunks", "firsts", "shorts"), lists)))

    def _table(self, step, T: int):
        """The step's cosines and sines, made by the first layer that turns by this rotation."""
        s = self.spec
        if s.rotary is None:
            return None
        key = ("rotation_table", s.rotary)
        table = step.shared.get(key)
        if table is None:
            n = sum(1 for k in step.shared if isinstance(k, tuple) and k[0] == "rotation_table")
            table = step.scratch(f"rotation_table{n}", (T, s.rotary.dims // 2, 2), torch.float32)
            ops.rotation_table(step.positions, self.freq, float(s.rotary.magnitude), table)
            step.shared[key] = table
        return table

    def inner(self, rows, out, step, cache) -> None:
        """From the rows [q | k | v | gate] of the input product to the gated heads."""
        s = self.spec
        T = rows.shape[0]
        QK, V = self.qk_width, self.v_width
        hints = step.hints.get(self.hint_key) if self.hint_key is not None else None
        lists = None
        if hints is not None and "chunks" in hints.arrays:
            lists = tuple(hints.arrays.get(n) for n in ("chunks", "firsts", "shorts"))
        o = step.scratch("rec_out", (T, V), torch.float32)
        ops.fixed_decay(rows[:, :QK], rows[:, QK:2 * QK], rows[:, 2 * QK:2 * QK + V], self.decay,
                        cache.state, step.state_slots, step.q_start, o, s.n_heads, s.head_dim,
                        s.value_dim, silu=s.silu, table=self._table(step, T),
                        k_scale=float(s.k_scale), lists=lists)
        ops.head_norm_gate(o, self.gain, rows[:, 2 * QK + V:2 * QK + 2 * V], out,
                           s.n_heads if s.norm == "head" else 1, float(s.norm_eps),
                           gate_kind=s.gate)

    def forward(self, h, residual, step, cache, accumulate: bool = True) -> None:
        T = h.shape[0]
        act = self.ctx.act_dtype
        if hasattr(h, "materialize"):
            h = h.materialize()
        rows = step.scratch("rec_proj", (T, self.proj.out_features), act)
        self.proj.forward(h, rows)
        mixed = step.scratch("rec_mixed", (T, self.v_width), act)
        self.inner(rows, mixed, step, cache)
        self.o.forward(mixed, residual, accumulate=accumulate, step=step if accumulate else None)


register_part("mixer", FixedDecayAttentionSpec, FixedDecayAttention)
