"""Mixers whose state is a matrix S [key size, value size] per head that keys and values write and queries read, in float32.

``gated_delta``: the delta rule with a decay per head and key channel (or per head alone).  q, k (``kv_heads`` heads), v pass a causal convolution
    per channel and silu; q and k heads are brought to unit length, q is multiplied by key_dim^(-1/2);
    g = exp(-exp(A_log) softplus(W_a2 W_a1 h + dt_bias)), beta = sigmoid(W_b h);
    S <- g S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q;   out = W_o (rms(o) * w * sigmoid(W_g2 W_g1 h)).
    ``decay="head"``: one decay per head, g = exp(-exp(A_log) softplus(W_a h + dt_bias)), and a dense gate, silu(W_g h).
``gated_linear_attention``: g = sigmoid(W_a2 W_a1 h + a2.b)^(1/tau) per head and key channel, no delta rule and no convolution:
    S <- g S + k v^T,  o = S^T q with q = W_q h key_dim^(-1/2);   out = W_o (rms(o) * w * silu(W_g h)).
``exponential_memory``: one decay per head from exponential gates.  i = cap tanh((W_i h + i.b) / cap), f = logsigmoid(cap
    tanh((W_f h + f.b) / cap)), a running maximum m <- max(f + m, i) that starts at zero;
    S <- exp(f + m' - m) S + exp(i - m) k v^T (m' the maximum before), n likewise with k alone;
    o = S^T q / (max(|n . q|, exp(-m)) + 1e-6);   out = W_o (rms(o) * w * sigmoid(W_g h)).
The norms over a head's o come before the weight: one of the head's size shared by the heads, or (``exponential_memory``) one
of all heads' size.  S, n, m and the convolution's inputs start at zero and live in one float32 row per request.

The projections that read h are rows of ONE product (the exponential gates have one of their own with a float32 result); the
second half of a low-rank decay is a product whose epilogue forms the factors (``ops.decay_product``; for many rows the
library's product with ``ops.decay_rows`` behind it); the recurrences
run in one kernel (``ops.matrix_memory``), the last step is ``ops.gated_head_norm``.
"""
import torch

from ..kernels import ops
from ..weights.loader import FreeDim, WeightSpec
from .base import CacheNeed, Mixer, packed_rows, register_part
from .linear import linear, linear_into_stream

UNIT_EPS = 1e-6            # under the root of the unit length of the delta rule's queries and keys
MAX_KEY_DIM = 1024         # rows of a head's state that the recurrence keeps in registers


def _check_sizes(what, heads, kv_heads, key_dim, value_dim):
    if heads <= 0 or kv_heads <= 0 or heads % kv_heads:
        raise ValueError("%s: %d heads are not a multiple of %d query/key heads" % (what, heads, kv_heads))
    if not 0 < key_dim <= MAX_KEY_DIM or not 0 < value_dim <= 1024:
        raise ValueError("%s: key and value sizes must lie in 1..1024 (got %d, %d)" % (what, key_dim, value_dim))


LIBRARY_ROWS = 256         # from so many tokens on the thin products (K an inner size) are the library's


class _MatrixMemory(Mixer):
    graph_safe = True
    relocatable = True
    adds_into_stream = True

    def cache_need(self):
        return CacheNeed("state", state_shape=((self.state_size + 3) // 4 * 4,), state_dtype=torch.float32)

    def _result(self, rows, ctx, into=None):
        if linear_into_stream(rows, self.w_o, into, ctx.ws, "mixer_tail", self.runtime.gemm_impl):
            return None
        y = ctx.ws.buffer(self.out_buffer, (rows.shape[0], self.hidden_size), self.runtime.dtype)
        linear(rows, self.w_o, y, self.runtime.gemm_impl, ws=ctx.ws)
        return y

    def _by_library(self, x):
        """Whether a thin product over the strided rows ``x`` goes to the library: many rows, whole 16-byte pieces."""
        piece = 16 // x.element_size()
        return x.shape[0] >= LIBRARY_ROWS and x.shape[1] % piece == 0 and x.stride(0) % piece == 0 and x.data_ptr() % 16 == 0

    def _decay(self, x, w, bias, ctx, **kind):
        """The decay factors, float32 [T, heads * key_dim], from the low-rank rows ``x``."""
        decay = ctx.ws.buffer("memory_decay", (x.shape[0], w.shape[0]), torch.float32)
        if not self._by_library(x):
            return ops.decay_product(x, w, decay, bias, **kind)
        linear(x, w, decay, self.runtime.gemm_impl, ws=ctx.ws)
        return ops.decay_rows(decay, bias, **kind)

    def _project(self, h, ctx):
        rows = ctx.ws.buffer("memory_rows", (h.shape[0], self.w_rows.shape[0]), self.runtime.dtype)
        linear(h, self.w_rows, rows, self.runtime.gemm_impl, ws=ctx.ws)
        return rows


@register_part("mixer", "gated_delta")
class GatedDeltaRule(_MatrixMemory):
    accepts_deferred = True

    def __init__(self, name, runtime, hidden_size: int, heads: int, kv_heads: int, key_dim: int, value_dim: int, conv_taps: int,
                 norm_eps: float, decay: str = "channel"):
        """``decay``: "channel" (low-rank decay and gate projections, a sigmoid gate) or "head" (dense ones, a silu gate)."""
        super().__init__(name, runtime)
        _check_sizes("gated delta rule", heads, kv_heads, key_dim, value_dim)
        if not 1 <= conv_taps <= 8:
            raise ValueError("gated delta rule: 1..8 convolution taps (got %d)" % conv_taps)
        if decay not in ("channel", "head"):
            raise ValueError("gated delta rule: the decay is per channel or per head (got %r)" % (decay,))
        self.per_head = decay == "head"
        self.hidden_size, self.heads, self.kvh = int(hidden_size), int(heads), int(kv_heads)
        self.dk, self.dv, self.taps, self.eps = int(key_dim), int(value_dim), int(conv_taps), float(norm_eps)
        self.nq, self.nv = self.kvh * self.dk, self.heads * self.dv
        self.channels = 2 * self.nq + self.nv                            # what passes the convolution: q, k, v
        self.conv_offset = self.heads * self.dv * self.dk                # the state: [S | the convolution's last inputs]
        self.state_size = self.conv_offset + (self.taps - 1) * self.channels
        self.ranks = (FreeDim(name + "a.rank", self.dk), FreeDim(name + "g.rank", self.dv))

    def _row_names(self):
        """What reads h, in the order of the packed projection's rows."""
        return ("q", "k", "v") + (("g", "b", "a") if self.per_head else ("a1", "g1", "b"))

    def weight_specs(self):
        n, d, (ra, rg) = self.name, self.hidden_size, self.ranks
        cpack = n + "conv.packed"
        conv = lambda c, i: WeightSpec((c, self.taps), "vector", pack=(cpack, i), mean=1.0 / self.taps)
        rows = {"q": self.nq, "k": self.nq, "v": self.nv, "b": self.heads, "a1": ra, "g1": rg, "g": self.nv, "a": self.heads}
        n_decays = self.heads if self.per_head else self.heads * self.dk
        specs = {n + x: WeightSpec((rows[x], d), pack=(n + "rows.packed", i)) for i, x in enumerate(self._row_names())}
        specs.update({
            n + "q.conv": conv(self.nq, 0), n + "k.conv": conv(self.nq, 1), n + "v.conv": conv(self.nv, 2),
            n + "A_log": WeightSpec((self.heads,), "vector", mean=0.0), n + "dt_bias": WeightSpec((n_decays,), "vector", mean=0.0),
            n + "norm": WeightSpec((self.dv,), "vector"), n + "o": WeightSpec((d, self.nv)),
        })
        if not self.per_head:
            specs[n + "a2"], specs[n + "g2"] = WeightSpec((self.heads * self.dk, ra)), WeightSpec((self.nv, rg))
        return specs

    def load_weights(self, tensors):
        n, dt = self.name, self.runtime.dtype
        self.w_rows = packed_rows(tensors, n + "rows.packed", [n + s for s in self._row_names()])
        self.conv_w = packed_rows(tensors, n + "conv.packed", [n + s + ".conv" for s in ("q", "k", "v")])
        if not self.per_head:
            self.ra, self.rg = tensors[n + "a2"].shape[1], tensors[n + "g2"].shape[1]
            self.w_a2, self.w_g2 = tensors[n + "a2"].to(dt).contiguous(), tensors[n + "g2"].to(dt).contiguous()
        self.rate = torch.exp(tensors[n + "A_log"].to(torch.float64)).to(torch.float32).contiguous()
        self.dt_bias, self.norm_w, self.w_o = tensors[n + "dt_bias"], tensors[n + "norm"], tensors[n + "o"]

    def _channel_parts(self, rows, ctx):
        """(the step sizes' rows, the decay factors, the gate's rows) from the low-rank rows."""
        rt, T, c = self.runtime, rows.shape[0], self.channels
        a1, g1 = rows[:, c:c + self.ra], rows[:, c + self.ra:c + self.ra + self.rg]
        decay = self._decay(a1, self.w_a2, self.dt_bias, ctx, rate=self.rate)
        gate = ctx.ws.buffer("memory_gate", (T, self.nv), rt.dtype)
        if self._by_library(g1):
            linear(g1, self.w_g2, gate, rt.gemm_impl, ws=ctx.ws)
        else:
            ops.blocked_product(g1.unsqueeze(1), self.w_g2.unsqueeze(0), gate.unsqueeze(1))
        return rows[:, c + self.ra + self.rg:], decay, gate

    def forward(self, h, ctx, cache, into=None):
        rt, T, c = self.runtime, h.shape[0], self.channels
        buf = ctx.ws.buffer
        rows = self._project(h, ctx)
        head_decay = None
        if self.per_head:
            gate, b, a = rows[:, c:c + self.nv], rows[:, c + self.nv:c + self.nv + self.heads], rows[:, c + self.nv + self.heads:]
            decay = buf("memory_decay", (T, self.heads), torch.float32)
            head_decay = (a, self.rate, self.dt_bias, decay)             # formed beside the step sizes
        else:
            b, decay, gate = self._channel_parts(rows, ctx)
        qkv, beta = buf("memory_qkv", (T, c), torch.float32), buf("memory_beta", (T, self.heads), torch.float32)
        single = ctx.T == ctx.R
        lists = (ctx.req_rows, ctx.state_slots, ctx.R)
        ops.delta_prep(rows[:, :c], self.conv_w, b, qkv, beta, self.kvh, self.heads, self.dk, self.dv, UNIT_EPS, cache.state,
                       self.state_base + self.conv_offset, ctx.token_req, *lists, single=single, head_decay=head_decay)
        o = buf("memory_o", (T, self.nv), torch.float32)
        ops.matrix_memory(qkv[:, :self.nq], qkv[:, self.nq:2 * self.nq], qkv[:, 2 * self.nq:], decay, self.heads, self.kvh, self.dk, self.dv,
                          o, cache.state, self.state_base, *lists, single=single, scale=beta, delta=True, q_scale=self.dk ** -0.5,
                          compute_units=ctx.cu_count)
        g = buf("memory_gated", (T, self.nv), rt.dtype)
        ops.gated_head_norm(o, gate, self.norm_w, self.heads, self.eps, g, gate="silu" if self.per_head else "sigmoid")
        return self._result(g, ctx, into)


@register_part("mixer", "gated_linear_attention")
class GatedLinearAttention(_MatrixMemory):
    accepts_deferred = True

    def __init__(self, name, runtime, hidden_size: int, heads: int, key_dim: int, value_dim: int, tau: float, norm_eps: float):
        super().__init__(name, runtime)
        _check_sizes("gated linear attention", heads, heads, key_dim, value_dim)
        if not float(tau) > 0:
            raise ValueError("gated linear attention: tau must be positive (got %r)" % (tau,))
        self.hidden_size, self.heads, self.dk, self.dv = int(hidden_size), int(heads), int(key_dim), int(value_dim)
        self.tau, self.eps = float(tau), float(norm_eps)
        self.nq, self.nv = self.heads * self.dk, self.heads * self.dv
        self.state_size = self.heads * self.dv * self.dk
        self.rank = FreeDim(name + "a.rank", 16)

    def weight_specs(self):
        n, d = self.name, self.hidden_size
        pack = n + "rows.packed"
        return {
            n + "q": WeightSpec((self.nq, d), pack=(pack, 0)), n + "k": WeightSpec((self.nq, d), pack=(pack, 1)),
            n + "v": WeightSpec((self.nv, d), pack=(pack, 2)), n + "g": WeightSpec((self.nv, d), pack=(pack, 3)),
            n + "a1": WeightSpec((self.rank, d), pack=(pack, 4)),
            n + "a2": WeightSpec((self.nq, self.rank)), n + "a2.b": WeightSpec((self.nq,), "vector", mean=0.0),
            n + "norm": WeightSpec((self.dv,), "vector"), n + "o": WeightSpec((d, self.nv)),
        }

    def load_weights(self, tensors):
        n = self.name
        self.w_rows = packed_rows(tensors, n + "rows.packed", [n + s for s in ("q", "k", "v", "g", "a1")])
        self.w_a2 = tensors[n + "a2"].to(self.runtime.dtype).contiguous()
        self.b_a2, self.norm_w, self.w_o = tensors[n + "a2.b"], tensors[n + "norm"], tensors[n + "o"]

    def forward(self, h, ctx, cache, into=None):
        rt, T, nq, nv = self.runtime, h.shape[0], self.nq, self.nv
        buf = ctx.ws.buffer
        rows = self._project(h, ctx)
        decay = self._decay(rows[:, 2 * nq + 2 * nv:], self.w_a2, self.b_a2, ctx, log_scale=1.0 / self.tau)
        o = buf("memory_o", (T, nv), torch.float32)
        ops.matrix_memory(rows[:, :nq], rows[:, nq:2 * nq], rows[:, 2 * nq:2 * nq + nv], decay, self.heads, self.heads, self.dk, self.dv, o,
                          cache.state, self.state_base, ctx.req_rows, ctx.state_slots, ctx.R, single=ctx.T == ctx.R,
                          q_scale=self.dk ** -0.5, compute_units=ctx.cu_count)
        g = buf("memory_gated", (T, nv), rt.dtype)
        ops.gated_head_norm(o, rows[:, 2 * nq + nv:2 * nq + 2 * nv], self.norm_w, self.heads, self.eps, g, gate="silu")
        return self._result(g, ctx, into)


@register_part("mixer", "exponential_memory")
class ExponentialMemory(_MatrixMemory):
    accepts_deferred = True

    def __init__(self, name, runtime, hidden_size: int, heads: int, key_dim: int, value_dim: int, gate_cap: float, norm_eps: float):
        super().__init__(name, runtime)
        _check_sizes("exponential memory", heads, heads, key_dim, value_dim)
        if not float(gate_cap) > 0:
            raise ValueError("exponential memory: the gates' cap must be positive (got %r)" % (gate_cap,))
        self.hidden_size, self.heads, self.dk, self.dv = int(hidden_size), int(heads), int(key_dim), int(value_dim)
        self.cap, self.eps = float(gate_cap), float(norm_eps)
        self.nq, self.nv = self.heads * self.dk, self.heads * self.dv
        self.max_offset = self.heads * (self.dv + 1) * self.dk           # the state: [S and n, a head's n behind its S | m]
        self.state_size = self.max_offset + self.heads

    def weight_specs(self):
        n, d = self.name, self.hidden_size
        pack, gpack = n + "rows.packed", n + "gates.packed"
        return {
            n + "q": WeightSpec((self.nq, d), pack=(pack, 0)), n + "k": WeightSpec((self.nq, d), pack=(pack, 1)),
            n + "v": WeightSpec((self.nv, d), pack=(pack, 2)), n + "g": WeightSpec((self.nv, d), pack=(pack, 3)),
            n + "i": WeightSpec((self.heads, d), pack=(gpack, 0)), n + "f": WeightSpec((self.heads, d), pack=(gpack, 1)),
            n + "i.b": WeightSpec((self.heads,), "vector", mean=0.0), n + "f.b": WeightSpec((self.heads,), "vector", mean=0.0),
            n + "norm": WeightSpec((self.nv,), "vector"), n + "o": WeightSpec((d, self.nv)),
        }

    def load_weights(self, tensors):
        n = self.name
        self.w_rows = packed_rows(tensors, n + "rows.packed", [n + s for s in ("q", "k", "v", "g")])
        self.w_gates = packed_rows(tensors, n + "gates.packed", [n + s for s in ("i", "f")])
        self.b_i, self.b_f = tensors[n + "i.b"], tensors[n + "f.b"]
        self.norm_w, self.w_o = tensors[n + "norm"], tensors[n + "o"]

    def forward(self, h, ctx, cache, into=None):
        rt, T, H, nq, nv = self.runtime, h.shape[0], self.heads, self.nq, self.nv
        buf = ctx.ws.buffer
        rows = self._project(h, ctx)
        z = buf("memory_gate_rows", (T, 2 * H), torch.float32)
        linear(h, self.w_gates, z, rt.gemm_impl, ws=ctx.ws)
        keep, add, floor, num = (buf("memory_" + s, (T, H), torch.float32) for s in ("keep", "add", "floor", "num"))
        lists = (ctx.req_rows, ctx.state_slots, ctx.R)
        ops.memory_gates(z, self.b_i, self.b_f, self.cap, keep, add, floor, cache.state, self.state_base + self.max_offset, *lists)
        o = buf("memory_o", (T, nv), torch.float32)
        ops.matrix_memory(rows[:, :nq], rows[:, nq:2 * nq], rows[:, 2 * nq:2 * nq + nv], keep, H, H, self.dk, self.dv, o, cache.state,
                          self.state_base, *lists, single=ctx.T == ctx.R, scale=add, q_scale=self.dk ** -0.5, extra_out=num,
                          compute_units=ctx.cu_count)
        g = buf("memory_gated", (T, nv), rt.dtype)
        ops.gated_head_norm(o, rows[:, 2 * nq + nv:], self.norm_w, H, self.eps, g, num=num, floor=floor)
        return self._result(g, ctx, into)
