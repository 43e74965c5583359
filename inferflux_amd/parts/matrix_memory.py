"""Matrix memory with exponential gates: a recurrence per head whose state is a matrix S [d, dv], decayed and written with one
number each per token, and a normaliser n [d] that is decayed and written alike.

With ``n_heads`` heads, queries and keys of ``head_dim`` channels and values of ``v_head_dim``, for a request's tokens:

    q = W_q h * head_dim^(-1/2),  k = W_k h,  v = W_v h,  g = W_g h
    i = cap tanh((W_i h + b_i) / cap),  f = log sigmoid(cap tanh((W_f h + b_f) / cap))      one of each per head, in float
    m_t = max(f + m_(t-1), i),  m_(-1) = 0                                                 the running maximum of the exponents
    S_t = exp(f + m_(t-1) - m_t) S_(t-1) + exp(i - m_t) k v^T,  S_(-1) = 0;  n_t likewise with k alone
    o_t = S_t^T q / (max(|n_t . q|, exp(-m_t)) + 1e-6)
    out = W_o ( rms(o_t) w_norm sigmoid(g) )            each head's o over its root mean square, a weight per channel of all heads

What a request carries from step to step is m, S and n: one float32 row of the engine's per-request state (``StateSpec``), laid
out as the kernels of ``csrc/matrix_memory.hip`` want it, zeroed when the request starts.  Nothing is kept per token, so the
layer owns no cache pages.  The gates' products give float32; q, k, v and g follow the activation type; everything behind
the projections is float.

Tensors (``tensors`` maps the roles "q", "k", "v", "g", "i", "f", "o", "i_bias", "f_bias", "norm" to full names; by default
``<name>.q_proj.weight`` and so on, ``<name>.i_proj.bias``, ``<name>.norm.weight`` [n_heads * v_head_dim]).
"""
from __future__ import annotations

from typing import Dict, Mapping, Optional

import torch

from ..kernels import ops
from .base import Mixer, MixerBinding, register_part
from .ffn import concat_weights
from .plan import ParamSpec, StateSpec


CHUNK_MIN_ROWS = 64         # a step that brings some request this many rows or more takes the chunks


@register_part("mixer", "matrix_memory")
class MatrixMemory(Mixer):
    graph_safe = True          # every kernel reads the step's layout from the context's device arrays
    adds_to_stream = True

    def __init__(self, name: str, hidden_size: int, n_heads: int, head_dim: int, v_head_dim: int, gate_cap: float, norm_eps: float,
                 init_std: float = 0.02, tensors: Optional[Mapping[str, str]] = None):
        self.name, self.hidden_size = name, int(hidden_size)
        self.n_heads, self.head_dim, self.v_head_dim = int(n_heads), int(head_dim), int(v_head_dim)
        self.gate_cap, self.norm_eps = float(gate_cap), float(norm_eps)
        if min(self.n_heads, self.head_dim, self.v_head_dim) <= 0 or self.gate_cap <= 0:
            raise ValueError(f"{name}: heads, head_dim, v_head_dim and gate_cap must be positive")
        ops.matrix_memory_layout(self.head_dim, self.v_head_dim)      # (refuses head sizes the kernel has no layout for)
        self.init_std = init_std
        self.names = {k: f"{name}.{k}_proj.weight" for k in ("q", "k", "v", "g", "i", "f", "o")}
        self.names.update({"i_bias": f"{name}.i_proj.bias", "f_bias": f"{name}.f_proj.bias", "norm": f"{name}.norm.weight"})
        self.names.update(tensors or {})
        self.qk_width, self.v_width = self.n_heads * self.head_dim, self.n_heads * self.v_head_dim
        self.w_in = self.w_main = self.w_gates = self.w_o = self.i_bias = self.f_bias = self.norm_w = None

    def state_spec(self) -> StateSpec:
        return StateSpec((ops.matrix_memory_state_floats(self.n_heads, self.head_dim, self.v_head_dim),), "float32")

    def param_specs(self) -> Dict[str, ParamSpec]:
        nm, H, s, nh = self.names, self.hidden_size, ("normal", self.init_std), self.n_heads
        QK, V = self.qk_width, self.v_width
        return {
            nm["q"]: ParamSpec((QK, H), s), nm["k"]: ParamSpec((QK, H), s), nm["v"]: ParamSpec((V, H), s), nm["g"]: ParamSpec((V, H), s),
            nm["i"]: ParamSpec((nh, H), s), nm["f"]: ParamSpec((nh, H), s), nm["i_bias"]: ParamSpec((nh,), ("uniform", -2.0, 2.0)),
            nm["f_bias"]: ParamSpec((nh,), ("uniform", 1.0, 6.0)), nm["o"]: ParamSpec((H, V), s), nm["norm"]: ParamSpec((V,), ("ones",)),
        }

    def load(self, tensors: Mapping[str, torch.Tensor]) -> None:
        nm = self.names
        stacked = concat_weights([tensors[nm[p]] for p in ("q", "k", "v", "g", "i", "f")])
        n = 2 * self.qk_width + 2 * self.v_width
        self.w_in = ops.prepare_linear(stacked)                       # q | k | v | g | i | f
        self.w_main, self.w_gates = self.w_in.part(0, n), self.w_in.part(n, n + 2 * self.n_heads)
        self.w_o = ops.prepare_linear(tensors[nm["o"]])
        wide = lambda k: tensors[nm[k]].float().contiguous()          # float whatever the file holds
        self.i_bias, self.f_bias, self.norm_w = wide("i_bias"), wide("f_bias"), wide("norm")

    def accepts_scaled_rows(self, n_rows: int) -> bool:
        return ops.takes_scaled_rows(n_rows, self.w_in)

    def forward(self, h, ctx, binding: MixerBinding, sink=None):
        state, t = binding.state, ctx.timer
        if state is None:
            raise ValueError(f"{self.name}: the mixer was given no per-request state")
        QK, V, nh, dtype = self.qk_width, self.v_width, self.n_heads, h.dtype
        # A prompt's portion walked token by token leaves most of the chip idle: in bfloat16 long portions are cut into chunks
        # that run side by side.  In 32-bit the walk stays in one piece, so that a token's sums do not depend on where its
        # request was cut.  (Steps of single tokens never take the chunks: a captured layout keeps its launches.)
        chunks = None
        if (ctx.n_tokens > ctx.n_requests and ops.matrix_memory_takes_chunks(dtype, self.head_dim, self.v_head_dim)
                and int(ctx.h_q_len.max()) >= CHUNK_MIN_ROWS):
            chunks = ctx.derived(("scan_chunks", ops.MEMORY_CHUNK),
                                 lambda: ops.scan_chunks(ctx.h_q_start, ctx.h_q_len, ops.MEMORY_CHUNK, ctx.device))
        if chunks is None and ops.streams_weight(h.shape[0], self.w_in):
            # few rows: one product whose float sums are read as they are
            rows = ops.linear(h, self.w_in, out_dtype=torch.float32)
            gates, i_col = rows, 2 * QK + 2 * V
        else:       # many rows: the activation type for what is wide, float for the gates
            rows = ops.linear(h, self.w_main)
            gates, i_col = ops.linear(h, self.w_gates, out_dtype=torch.float32), 0
        if t is not None:
            t.mark("mixer.project")
        y = ops.matrix_memory(rows, (0, QK, 2 * QK, 2 * QK + V), gates, (i_col, i_col + nh), self.i_bias, self.f_bias, self.gate_cap,
                              self.norm_w, self.norm_eps, nh, self.head_dim, self.v_head_dim, state, ctx.q_start, ctx.q_len,
                              ctx.state_slots, ctx.row_req, dtype, single_tokens=ctx.n_tokens == ctx.n_requests, chunks=chunks)
        if t is not None:
            t.mark("mixer.scan")
        if sink is not None and ops.adds_into_stream(y.shape[0], self.w_o, sink.norm_weight):
            return ops.linear_into_stream(y, self.w_o, sink.stream, sink.norm_weight, sink.eps, sink.mult)
        return ops.linear(y, self.w_o, keep_slices=sink is not None)
