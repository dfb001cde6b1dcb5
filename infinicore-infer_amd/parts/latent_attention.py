"""Softmax attention through a latent: queries, keys and values are made from low-rank vectors, and only the
key/value latent c (``kv_rank`` values, RMS-normed) and one rotated key part shared by all heads (``rot_dim`` values) are
cached per token, as ONE row of a single-plane paged cache.

    c_q = norm(W_dq h),  q = W_uq c_q = per head [dim plain | rot_dim rotated]
    W_dkv h = [kv_rank -> c = norm(.) | rot_dim -> k_rot, rotated, not normed]
    k_h = W_uk,h c,  v_h = W_uv,h c,  s = scale (q_plain . k_h + q_rot . k_rot),  causal softmax,
    out = W_o (concat_h(sum_j p_j v_hj) * sigmoid(W_g h))            (the gate is optional)

Options, each a parameter: a window (query i sees key j when 0 <= i - j < window), a learned sink per head in the softmax's
denominator (the tensor ``sink``), stretched wavelengths of the rotation (``parts/rotary.py``), and ``own_rows=False``: the layer
has no W_dkv and reads the rows that another entry of the run order cached.

Single tokens (and short portions): the keys and values are never made.  With q' = W_uk,h^T q_plain the score is
q' . c + q_rot . k_rot and the head's result is W_uv,h (sum_j p_j c_j), so every head walks the same cached rows and two small
products per head stand before and after the walk.  Prompt portions in bfloat16 make keys and values per head from the
request's gathered rows with one product and walk those (a third of the arithmetic at a portion's length), where the kernel has
the sizes; otherwise two matrix products over the latent rows.  Rotation: pairs (2i, 2i+1) of the first ``rot_dims`` entries of a
rotated part turn by position * f_i, computed in float32.
"""
import torch

from ..kernels import ops
from ..weights.loader import FreeDim, WeightSpec
from .base import CacheNeed, Mixer, packed_rows, register_part
from .linear import _library, linear, linear_into_stream
from .rotary import pair_frequencies, stretched_magnitude

PORTION_MIN = 32                       # tokens from which a portion makes keys and values per head
MADE_KEYS_BYTES = 8 << 30              # most memory the keys and values made for one portion may take


@register_part("mixer", "latent_attention")
class LatentAttention(Mixer):
    graph_safe = True
    accepts_deferred = True
    adds_into_stream = True

    def __init__(self, name, runtime, hidden_size: int, num_heads: int, head_dim: int, rot_dim: int, value_dim: int,
                 q_rank, kv_rank: int, softmax_scale: float, rot_base: float, rot_dims=None, norm_eps: float = 1e-6,
                 gate: bool = True, window=None, sink: bool = False, rot_scaling=None, own_rows: bool = True):
        """``q_rank`` None: the tensors decide the query latent's size."""
        super().__init__(name, runtime)
        rot_dims = rot_dim if rot_dims is None else int(rot_dims)
        if min(num_heads, head_dim, value_dim, 1 if q_rank is None else q_rank, kv_rank) <= 0 or rot_dim < 0:
            raise ValueError("latent attention: sizes must be positive")
        if kv_rank > ops.LATENT_MAX_RANK:
            raise ValueError("latent attention: a latent of %d values is beyond the kernel's %d" % (kv_rank, ops.LATENT_MAX_RANK))
        if rot_dims % 2 or not 0 <= rot_dims <= rot_dim:
            raise ValueError("latent attention: %d rotated dimensions do not fit a rotated part of %d" % (rot_dims, rot_dim))
        if window is not None and int(window) <= 0:
            raise ValueError("latent attention: the window must be positive (got %r)" % (window,))
        self.hidden_size, self.H, self.dim, self.E, self.dv = int(hidden_size), int(num_heads), int(head_dim), int(rot_dim), int(value_dim)
        self.Rq, self.R = None if q_rank is None else int(q_rank), int(kv_rank)
        self.scale, self.eps, self.gate = float(softmax_scale), float(norm_eps), bool(gate)
        self.window, self.sink, self.own_rows = int(window) if window else 0, bool(sink), bool(own_rows)
        self.rot_dims = rot_dims
        self.freq = pair_frequencies(max(rot_dims, 2), rot_base, rot_scaling).to(runtime.device)
        self.rot_mult = stretched_magnitude(rot_scaling)
        self.sinks = self.kvn_w = None

    def cache_need(self):
        return CacheNeed("kv", n_kv_heads=1, head_dim=self.R + self.E, window=self.window or None, planes=1)

    def weight_specs(self):
        n, d, H = self.name, self.hidden_size, self.H
        pack = n + "down.packed"
        Rq = FreeDim(n + "q.rank", max(1, d // 3)) if self.Rq is None else self.Rq
        specs = {
            n + "dq": WeightSpec((Rq, d), pack=(pack, 0)),
            n + "dq.norm": WeightSpec((Rq,), "vector"),
            n + "uq": WeightSpec((H * (self.dim + self.E), Rq)),
            n + "uk": WeightSpec((H * self.dim, self.R), pack=(n + "ukv.packed", 0)),
            n + "uv": WeightSpec((H * self.dv, self.R), pack=(n + "ukv.packed", 1)),
            n + "o": WeightSpec((d, H * self.dv)),
        }
        if self.own_rows:
            specs[n + "dkv"] = WeightSpec((self.R + self.E, d), pack=(pack, 1))
            specs[n + "dkv.norm"] = WeightSpec((self.R,), "vector")
        if self.sink:
            specs[n + "sink"] = WeightSpec((self.H,), "vector", mean=0.0)
        if self.gate:
            specs[n + "g"] = WeightSpec((H * self.dv, d), pack=(pack, 2))
        return specs

    def load_weights(self, tensors):
        n, H = self.name, self.H
        self.w_down = packed_rows(tensors, n + "down.packed",
                                  [n + x for x, there in (("dq", True), ("dkv", self.own_rows), ("g", self.gate)) if there])
        self.qn_w = tensors[n + "dq.norm"]
        self.Rq = self.qn_w.shape[0]
        if self.own_rows:
            self.kvn_w = tensors[n + "dkv.norm"]
        if self.sink:
            self.sinks = tensors[n + "sink"].to(torch.float32).contiguous()
        self.w_uq, self.w_o = tensors[n + "uq"], tensors[n + "o"]
        # per head: W_uk^T [kv_rank, dim] takes a plain query into the latent's space; W_uv [value_dim, kv_rank] takes the walk's result out
        dt = self.runtime.dtype
        self.w_uk_t = tensors[n + "uk"].view(H, self.dim, self.R).transpose(1, 2).to(dt).contiguous()
        self.w_ukv = packed_rows(tensors, n + "ukv.packed", [n + "uk", n + "uv"]).to(dt)      # keys and values made from latent rows: one product
        self.w_uv = self.w_ukv[H * self.dim:].view(H, self.dv, self.R)

    def _key_splits(self, ctx, n_rows: int, most_keys: int) -> int:
        """Ways to split the keys of rows that walk the cache one by one, so that few rows still fill the chip: a function of
        the step's shape (such rows, rounded key count) alone."""
        if not n_rows or not most_keys:
            return 1
        if self.window:
            most_keys = min(most_keys, self.window + 31)
        on_cores = ops.attention_latent_on_matrix_cores(self.runtime.dtype, self.R, self.E)
        blocks = n_rows * ((self.H + 31) // 32 if on_cores else (self.H + 3) // 4)
        steps = (most_keys + 31) // 32 if on_cores else (most_keys + 63) // 64
        return max(1, min(32, steps // 2, (2 * ctx.cu_count + blocks - 1) // blocks))

    def _plan(self, ctx, T: int):
        """(runs of rows that walk the cache one by one as (first row, rows, most keys), portions that take matrix products as
        (batch row, first row, tokens, first position)).  A pure decode step is one run, whatever the positions are."""
        if T == ctx.R:
            return [(0, T, ctx.max_context)], []
        if self.runtime.dtype != torch.bfloat16 or self.runtime.attention_impl != "auto":
            return [(0, T, 0)], []
        least = PORTION_MIN if self._makes_keys() else 2
        runs, portions = [], []
        for r, n in enumerate(ctx.req_len):
            row0, pos0 = ctx.req_start[r], ctx.req_pos[r]
            if n >= least:
                portions.append((r, row0, n, pos0))
                continue
            most = ops.rule_context_bucket(pos0 + n)
            if runs and runs[-1][0] + runs[-1][1] == row0:
                runs[-1] = (runs[-1][0], runs[-1][1] + n, max(runs[-1][2], most))
            else:
                runs.append((row0, n, most))
        return runs, portions

    def _makes_keys(self) -> bool:
        return self.scale > 0 and self.R % 8 == 0 and ops.attention_latent_prefill_supported(self.runtime.dtype, self.dim, self.E, self.dv)

    def _walk(self, run, q, gate, heads_out, ctx, cache):
        """Rows that walk the cached rows one by one: queries into the latent's space, the walk, the heads' values out of it."""
        rt, H, R, E = self.runtime, self.H, self.R, self.E
        row0, n, most_keys = run
        rows = slice(row0, row0 + n)
        q = q[rows]
        qa = ctx.ws.buffer("latent_qa", (n, H * (R + E)), rt.dtype)
        ops.blocked_product(q.view(n, H, self.dim + E)[:, :, :self.dim], self.w_uk_t, qa.view(n, H, R + E)[:, :, :R])
        ops.latent_q_rotate(q, self.dim, E, R, H, self.freq, self.rot_dims, ctx.positions[rows], qa, self.rot_mult)
        walked = ctx.ws.buffer("latent_walk", (n, H * R), rt.dtype)
        n_split = self._key_splits(ctx, n, most_keys)
        part_acc = part_ml = None
        if n_split > 1:
            part_acc = ctx.ws.buffer("latent_part_acc", (n * H * n_split * R,), torch.float32)
            part_ml = ctx.ws.buffer("latent_part_ml", (n * H * n_split * 2,), torch.float32)
        ops.attention_latent(qa, walked, cache.k, cache.block_tables, ctx.token_req[rows], ctx.positions[rows], H, R, E, ctx.page_size,
                             self.scale, n_split, part_acc, part_ml, window=self.window, sinks=self.sinks)
        ops.blocked_product(walked.view(n, H, R), self.w_uv, heads_out[rows].view(n, H, self.dv),
                            gate=None if gate is None else gate[rows].view(n, H, self.dv))

    def _portion_by_keys(self, portion, q, gate, heads_out, ctx, cache) -> bool:
        """A portion over keys and values made per head from the request's rows (q's rotated parts are turned in place)."""
        r, row0, n, pos0 = portion
        H, R, D = self.H, self.R, self.R + self.E
        first = max(0, pos0 - self.window + 1) if self.window else 0
        key0, L = first // 16 * 16, pos0 + n
        keys = (L - key0 + 15) // 16 * 16
        width = self.w_ukv.shape[0]
        if 2 * keys * width > MADE_KEYS_BYTES:
            return False
        gathered = ctx.ws.buffer("latent_gathered", (keys, D), self.runtime.dtype)
        ops.latent_gather(cache.k, cache.block_tables[r], L, keys, ctx.page_size, R, gathered, key0=key0, first=first)
        kv = ctx.ws.buffer("latent_made", (keys, width), self.runtime.dtype)
        _library(gathered[:, :R], self.w_ukv, kv)
        mine = q[row0:row0 + n]
        ops.latent_q_rotate(mine, self.dim, self.E, self.dim, H, self.freq, self.rot_dims, ctx.positions[row0:row0 + n], mine, self.rot_mult)
        ops.attention_latent_prefill(q, heads_out, gate, kv, gathered, R, key0, row0, n, pos0, H, self.dim, self.E, self.dv, self.scale,
                                     window=self.window, sinks=self.sinks)
        return True

    def _portion_by_products(self, portion, q, gate, heads_out, ctx, cache):
        """A portion as two matrix products over all its (token, head) rows and the request's latent rows."""
        rt, H, R, E, D = self.runtime, self.H, self.R, self.E, self.R + self.E
        r, row0, n, pos0 = portion
        rows, L = slice(row0, row0 + n), pos0 + n
        qa = ctx.ws.buffer("latent_qa", (n, H * D), rt.dtype)
        ops.blocked_product(q[rows].view(n, H, self.dim + E)[:, :, :self.dim], self.w_uk_t, qa.view(n, H, D)[:, :, :R])
        ops.latent_q_rotate(q[rows], self.dim, E, R, H, self.freq, self.rot_dims, ctx.positions[rows], qa, self.rot_mult)
        walked = ctx.ws.buffer("latent_walk", (n, H * R), rt.dtype)
        first = max(0, pos0 - self.window + 1) if self.window else 0
        key0 = first // 16 * 16
        keys = (L - key0 + 15) // 16 * 16
        gathered = ctx.ws.buffer("latent_gathered", (keys, D), rt.dtype)
        gathered_t = ctx.ws.buffer("latent_gathered_t", (R, keys), rt.dtype)
        ops.latent_gather(cache.k, cache.block_tables[r], L, keys, ctx.page_size, R, gathered, gathered_t, key0=key0, first=first)
        per = max(1, min(n, (32 << 20) // (H * keys)))          # tokens per pass: the scores of a pass stay under 128 MB
        if self.window:
            per = min(per, max(self.window, 64))                # (and most of a pass's scores are seen)
        for q0 in range(0, n, per):
            qn = min(per, n - q0)
            # keys before the pass's first window and beyond its last token are not computed
            c0 = max(0, pos0 + q0 - self.window + 1) // 16 * 16 - key0 if self.window else 0
            cols = min(keys, (pos0 + q0 + qn - key0 + 15) // 16 * 16) - c0
            scores = ctx.ws.buffer("latent_scores", (qn * H, cols), torch.float32)
            _library(qa[q0:q0 + qn].view(qn * H, D), gathered[c0:c0 + cols], scores)
            probs = ctx.ws.buffer("latent_probs", (qn * H, cols), rt.dtype)
            ops.latent_softmax(scores, probs, H, pos0 + q0, self.scale, window=self.window, sinks=self.sinks, key0=key0 + c0)
            _library(probs, gathered_t[:, c0:c0 + cols], walked[q0:q0 + qn].view(qn * H, R))
        ops.blocked_product(walked.view(n, H, R), self.w_uv, heads_out[rows].view(n, H, self.dv),
                            gate=None if gate is None else gate[rows].view(n, H, self.dv))

    def forward(self, h, ctx, cache, into=None):
        rt, T, H, R, E = self.runtime, h.shape[0], self.H, self.R, self.E
        rows = ctx.ws.buffer("latent_rows", (T, self.w_down.shape[0]), rt.dtype)
        linear(h, self.w_down, rows, rt.gemm_impl, ws=ctx.ws)
        cq = ctx.ws.buffer("latent_cq", (T, self.Rq), rt.dtype)
        ops.latent_prep(rows, self.Rq, R, E, self.qn_w, self.kvn_w, self.eps, self.freq, self.rot_dims, ctx.positions, cq,
                        cache.k, cache.slots if cache.writes and self.own_rows else None, self.rot_mult)
        q = ctx.ws.buffer("latent_q", (T, H * (self.dim + E)), rt.dtype)
        linear(cq, self.w_uq, q, rt.gemm_impl, ws=ctx.ws)
        heads_out = ctx.ws.buffer("latent_heads", (T, H * self.dv), rt.dtype)
        gate = rows[:, rows.shape[1] - H * self.dv:] if self.gate else None
        runs, portions = self._plan(ctx, T)
        for run in runs:
            self._walk(run, q, gate, heads_out, ctx, cache)
        for portion in portions:
            if not (self._makes_keys() and self._portion_by_keys(portion, q, gate, heads_out, ctx, cache)):
                self._portion_by_products(portion, q, gate, heads_out, ctx, cache)
        if linear_into_stream(heads_out, self.w_o, into, ctx.ws, "mixer_tail", rt.gemm_impl):
            return None
        y = ctx.ws.buffer("mixer_out", (T, self.hidden_size), rt.dtype)
        linear(heads_out, self.w_o, y, rt.gemm_impl, ws=ctx.ws)
        return y
