"""Mixers side by side: all read the same input, the result is the sum of theirs, each times a constant.

At most one of them walks a paged cache; their states lie one after the other in the slot's state row (every mixer is told
where its own begins), and each writes its result to a buffer of its own."""
from dataclasses import replace

from .base import Branches, CacheNeed, Mixer, build_part, register_part


@register_part("mixer", "parallel")
class ParallelMixers(Mixer):
    graph_safe = True
    yields_branches = True

    def __init__(self, name, runtime, branches):
        """``branches``: one or two (mixer's PartSpec, factor)."""
        super().__init__(name, runtime)
        if not 1 <= len(branches) <= 2:
            raise ValueError("parallel mixers: one or two branches (got %d)" % len(branches))
        self.children = [build_part("mixer", spec, runtime) for spec, _ in branches]
        self.factors = [float(f) for _, f in branches]
        base = 0
        for i, c in enumerate(self.children):
            if not c.relocatable:
                raise ValueError("parallel mixers: %s keeps its state and result at fixed places" % type(c).__name__)
            c.state_base, c.out_buffer = base, "mixer_out_%d" % i
            need = c.cache_need()
            if need.has_state:
                if len(need.state_shape) != 1:
                    raise ValueError("parallel mixers: %s keeps a state that is no row of numbers" % type(c).__name__)
                base += (need.state_shape[0] + 3) // 4 * 4           # every state starts on 16 bytes
        self.state_size = base
        self.accepts_deferred = all(c.accepts_deferred for c in self.children)
        self.adds_into_stream = any(c.adds_into_stream for c in self.children)
        self._need = self._joined_need()

    def _joined_need(self) -> CacheNeed:
        needs = [c.cache_need() for c in self.children]
        paged = [n for n in needs if n.paged]
        states = {n.state_dtype for n in needs if n.has_state}
        if len(paged) > 1 or len(states) > 1:
            raise ValueError("parallel mixers: one paged cache and one kind of state at most")
        shape = (self.state_size,) if self.state_size else ()
        if not paged:
            return CacheNeed("state", state_shape=shape, state_dtype=states.pop()) if shape else CacheNeed()
        p = paged[0]
        kw = dict(state_shape=shape, state_dtype=states.pop()) if shape else {}
        return CacheNeed("kv+state" if shape else "kv", p.n_kv_heads, p.head_dim, p.window, planes=p.planes, plane_dims=p.plane_dims,
                         keep_first=p.keep_first, block_rows=p.block_rows, **kw)

    def sub_parts(self):
        return tuple(self.children)

    def cache_need(self):
        return self._need

    def forward(self, h, ctx, cache, branches: bool = False, into=None):
        parts = []
        for c, f in zip(self.children, self.factors):
            # a child that adds its result to the stream by itself does so with its factor
            mine = None if into is None or not c.adds_into_stream else replace(into, alpha=into.alpha * f)
            y = c.forward(h, ctx, cache) if mine is None else c.forward(h, ctx, cache, into=mine)
            if y is not None:
                parts.append((y, f))
        out = Branches(tuple(parts))
        if branches:
            return out
        if not parts:
            return None
        y = ctx.ws.buffer("mixer_out", tuple(out.parts[0][0].shape), self.runtime.dtype)
        y.zero_()
        for v, f in out.parts:
            y.add_(v, alpha=f)
        return y
