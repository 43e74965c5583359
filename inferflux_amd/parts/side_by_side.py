"""Several mixers over the same rows, their outputs added with a factor each: out = sum_i scale_i mixer_i(h).

Each part is built as it would be alone and works on its own part of the binding.  At most one of them keeps keys and values
and at most one keeps per-request state (a schedule entry owns one cache and one state).  In steps of few rows a part may add
its output, times its factor, to the stream itself; otherwise the outputs travel on as one ``DeltaSum``.
"""
from __future__ import annotations

import dataclasses
from typing import Sequence

from ..kernels.ops import DeltaSum, ScaledRows
from .base import Mixer, MixerBinding, build_part, register_part
from .plan import PartSpec


@register_part("mixer", "side_by_side")
class SideBySideMixers(Mixer):
    adds_to_stream = True
    graph_safe = True          # (of its own work; the parts say so of theirs)

    def __init__(self, name: str, hidden_size: int, mixers: Sequence[PartSpec], scales: Sequence[float]):
        if len(mixers) != len(scales) or not mixers:
            raise ValueError(f"{name}: {len(mixers)} mixers with {len(scales)} factors")
        self.name = name
        self.mixers = tuple(build_part("mixer", m, hidden_size=hidden_size) for m in mixers)
        self.scales = tuple(float(s) for s in scales)
        if sum(m.cache_spec() is not None for m in self.mixers) > 1 or sum(m.state_spec() is not None for m in self.mixers) > 1:
            raise ValueError(f"{name}: at most one of the mixers side by side may keep keys and values, and at most one state")

    def children(self):
        return self.mixers

    def cache_spec(self):
        return next((s for s in (m.cache_spec() for m in self.mixers) if s is not None), None)

    def state_spec(self):
        return next((s for s in (m.state_spec() for m in self.mixers) if s is not None), None)

    def accepts_scaled_rows(self, n_rows: int) -> bool:
        return all(m.accepts_scaled_rows(n_rows) for m in self.mixers)

    def forward(self, h, ctx, binding: MixerBinding, sink=None):
        terms, last = [], None
        for m, scale in zip(self.mixers, self.scales):
            mine = MixerBinding(cache=binding.cache if m.cache_spec() is not None else None, writes_cache=binding.writes_cache,
                                state=binding.state if m.state_spec() is not None else None)
            if sink is not None and m.adds_to_stream:
                out = m.forward(h, ctx, mine, sink=dataclasses.replace(sink, mult=sink.mult * scale))
            else:
                out = m.forward(h, ctx, mine)
            if isinstance(out, ScaledRows):
                last = out                       # (in the stream, with its factor)
            else:
                terms.append((out, scale))
        return DeltaSum(terms) if terms else last
