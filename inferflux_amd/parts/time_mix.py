"""Time mixing: a recurrence per head whose state is a matrix S [d, d], with a decay per key channel and token and a bonus for
the current token, fed by mixes of each row with the row before it.

With ``n_heads`` heads of ``head_dim`` channels for keys and values alike and a decay projected through ``decay_rank`` numbers,
for a request's rows h_0, h_1, ... (h_(-1) = 0):

    x_s = h_t + (h_(t-1) - h_t) mu_s                       for s of r, k, v, g, w
    r, k, v, g = W_r x_r, W_k x_k, W_v x_v, W_g x_g
    w = exp(-exp(W_w2 tanh(W_w1 x_w) + w0))                per head and key channel, in float
    o_t = (S_(t-1) + diag(u) k_t v_t^T)^T r_t              per head, in float
    S_t = diag(w_t) S_(t-1) + k_t v_t^T,  S_(-1) = 0
    out = W_o ( rms(o_t) w_norm silu(g) )                  each head's o over its root mean square, a weight per channel of all heads

What a request carries from step to step is its last row h and its S: one float32 row of the engine's per-request state
(``StateSpec``), the last row first, S laid out as the kernel of ``csrc/gla.hip`` wants it, zeroed when the request starts.
Nothing is kept per token, so the layer owns no cache pages.

Tensors (``tensors`` maps the roles "r", "k", "v", "g", "o", "w1", "w2", "w0", "u", "norm", "mu_r" ... "mu_w" to full names; by
default ``<name>.r_proj.weight`` and so on, ``<name>.w1``, ``<name>.w2``, ``<name>.w0``, ``<name>.u`` [n_heads, head_dim],
``<name>.norm.weight`` [n_heads * head_dim], ``<name>.mu_r``).
"""
from __future__ import annotations

from typing import Dict, Mapping, Optional

import torch

from ..kernels import ops
from .base import Mixer, MixerBinding, register_part
from .ffn import concat_weights
from .gla import SCAN_CHUNK, SCAN_CHUNK_MIN_ROWS
from .plan import ParamSpec, StateSpec

SOURCES = ("r", "k", "v", "g", "w")        # the order of the mixes, and of the projections that read them


@register_part("mixer", "time_mix")
class TimeMix(Mixer):
    graph_safe = True          # every kernel reads the step's layout from the context's device arrays
    adds_to_stream = True

    def __init__(self, name: str, hidden_size: int, n_heads: int, head_dim: int, decay_rank: int, norm_eps: float,
                 init_std: float = 0.02, tensors: Optional[Mapping[str, str]] = None):
        self.name, self.hidden_size = name, int(hidden_size)
        self.n_heads, self.head_dim, self.decay_rank, self.norm_eps = int(n_heads), int(head_dim), int(decay_rank), float(norm_eps)
        if min(self.n_heads, self.head_dim, self.decay_rank) <= 0:
            raise ValueError(f"{name}: heads, head_dim and decay_rank must be positive")
        ops.gla_layout(self.head_dim, self.head_dim)            # (refuses head sizes the kernel has no layout for)
        self.init_std = init_std
        self.names = {k: f"{name}.{k}_proj.weight" for k in ("r", "k", "v", "g", "o")}
        self.names.update({k: f"{name}.{k}" for k in ("w1", "w2", "w0", "u")})
        self.names.update({f"mu_{s}": f"{name}.mu_{s}" for s in SOURCES})
        self.names["norm"] = f"{name}.norm.weight"
        self.names.update(tensors or {})
        self.width = self.n_heads * self.head_dim
        self.shift_floats = -(-self.hidden_size // 4) * 4       # the last row's part of a state row comes first
        self.w_each = self.w_all = self.w2 = self.w_o = self.w0 = self.u = self.mu = self.norm_w = None

    def state_spec(self) -> StateSpec:
        return StateSpec((self.shift_floats + ops.gla_state_floats(self.n_heads, self.head_dim, self.head_dim),), "float32")

    def param_specs(self) -> Dict[str, ParamSpec]:
        nm, H, W, s = self.names, self.hidden_size, self.width, ("normal", self.init_std)
        out = {nm[k]: ParamSpec((W, H), s) for k in ("r", "k", "v", "g")}
        out.update({nm[f"mu_{k}"]: ParamSpec((H,), ("uniform", 0.0, 1.0)) for k in SOURCES})
        out.update({nm["o"]: ParamSpec((H, W), s), nm["w1"]: ParamSpec((self.decay_rank, H), s),
                    nm["w2"]: ParamSpec((W, self.decay_rank), ("normal", 0.1)), nm["w0"]: ParamSpec((W,), ("uniform", -5.0, 0.0)),
                    nm["u"]: ParamSpec((self.n_heads, self.head_dim), ("normal", 0.5)), nm["norm"]: ParamSpec((W,), ("ones",))})
        return out

    def load(self, tensors: Mapping[str, torch.Tensor]) -> None:
        nm = self.names
        stacked = concat_weights([tensors[nm[p]] for p in ("r", "k", "v", "g", "w1")])
        W = self.width
        self.w_all = ops.prepare_linear(stacked, tile_rows=16)       # r | k | v | g | w1, for few rows: one product over five inputs
        self.w_each = [self.w_all.part(i * W, (i + 1) * W) for i in range(4)] + [self.w_all.part(4 * W, 4 * W + self.decay_rank)]
        self.w2 = tensors[nm["w2"]].t().contiguous()                 # [rank, width]: neighbouring lanes read neighbouring channels
        self.w_o = ops.prepare_linear(tensors[nm["o"]])
        wide = lambda k: tensors[nm[k]].float().contiguous()         # float whatever the file holds
        self.w0, self.u, self.norm_w = wide("w0"), wide("u"), wide("norm")
        self.mu = torch.stack([wide(f"mu_{s}") for s in SOURCES]).contiguous()

    def _project(self, x):
        """(r, k, v, g) [T, width] each and the decay's inner product [T, rank] (float) of the five mixes x [5, T, H]."""
        if ops.takes_blocks(x.shape[1], self.w_all, self.width):
            rows = ops.linear_blocks(x, self.w_all, self.width, torch.float32)
            W = self.width
            return [rows[:, i * W:(i + 1) * W] for i in range(4)], rows[:, 4 * W:]
        return [ops.linear(x[i], self.w_each[i]) for i in range(4)], ops.linear(x[4], self.w_each[4], out_dtype=torch.float32)

    def forward(self, h, ctx, binding: MixerBinding, sink=None):
        state, t = binding.state, ctx.timer
        if state is None:
            raise ValueError(f"{self.name}: the mixer was given no per-request state")
        x = ops.shifted_mixes(h, self.mu, state, 0, ctx.row_req, ctx.q_start, ctx.q_len, ctx.state_slots)
        (r, k, v, g), a = self._project(x)
        z = ops.lowrank_tanh(a, self.w2)                        # the decay's second product: its logits are never rounded
        if t is not None:
            t.mark("mixer.project")
        # (long portions in chunks that run side by side in bfloat16, one walk in 32-bit: as gated linear attention has it)
        chunks = None
        if h.dtype == torch.bfloat16 and ctx.n_tokens > ctx.n_requests and int(ctx.h_q_len.max()) >= SCAN_CHUNK_MIN_ROWS:
            chunks = ctx.derived(("scan_chunks", SCAN_CHUNK), lambda: ops.scan_chunks(ctx.h_q_start, ctx.h_q_len, SCAN_CHUNK, ctx.device))
        y = ops.time_mix_scan(r, k, v, g, z, self.w0, self.u, self.norm_w, self.norm_eps, self.n_heads, self.head_dim, state,
                              self.shift_floats, ctx.q_start, ctx.q_len, ctx.state_slots, h.dtype, chunks)
        if t is not None:
            t.mark("mixer.scan")
        if sink is not None and ops.adds_into_stream(y.shape[0], self.w_o, sink.norm_weight):
            return ops.linear_into_stream(y, self.w_o, sink.stream, sink.norm_weight, sink.eps, sink.mult)
        return ops.linear(y, self.w_o, keep_slices=sink is not None)
