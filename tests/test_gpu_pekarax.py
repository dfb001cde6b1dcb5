"""The Pekarax decoder in the engine against the plain implementation of its equations (plain_pekarax.py): each
mechanism's kernel alone, then whole models in the four replay modes and both dtypes, with sizes, counts, constants and
layer orders that differ from model to model, and greedy generation through the entry point."""
import json
import math
import os
import random

import pytest
import torch

import helpers as H
import plain_pekarax as P

pytestmark = pytest.mark.gpu

DTYPES = [("float32", torch.float32, 2e-4), ("bfloat16", torch.bfloat16, 8e-2)]
BF16_MEAN = 4e-2
BF16_MEDIAN = 2e-2


def _compare(got, ref, dtype, tol, what, steps=None, rounded=None):
    """float32: every position within ``tol`` of the largest logit (with ``rounded``, for configurations drawn at random: all
    but one in a hundred, and none beyond five times that; a position where values nearly cancel before a norm magnifies
    rounding).  bfloat16: the median and the mean over positions, and all but a few positions within ``tol``: where two
    experts' scores lie closer than 16-bit rounding the choice may fall the other way and move that token's row and, through
    a recurrent state, those behind it (every position is held to the float32 tolerance in the float32 mode, which runs the
    same steps, and the 16-bit kernels are held to theirs one by one).  ``rounded``: the plain implementation's logits with the
    sublayers' inputs and results rounded to 16 bits; the median must then stay within three
    times what that moves (the mean, which a single flipped choice can carry, too if that is more than its own bound)."""
    if dtype == torch.float32 and rounded is None:
        return H.compare(got, ref, tol, what, steps)
    H.compare(got, ref, 5 * tol if dtype == torch.float32 else 1e9, what, steps)        # every wanted place is there and finite
    error = lambda rid, pos, row: float((row.double() - ref[rid][pos]).abs().max()) / float(ref[rid].abs().max())
    errs = sorted(error(rid, pos, row) for (rid, pos), row in got.items())
    n, middle = len(errs), errs[len(errs) // 2]
    over = sum(e > tol for e in errs)
    if dtype == torch.float32:
        assert over <= max(1, 0.01 * n), "%s: %d of %d positions beyond %.3g" % (what, over, n, tol)
        return errs[-1], None
    median_most, mean_most, over_most = BF16_MEDIAN, BF16_MEAN, max(1, 0.15 * n)
    if rounded is not None:
        alone = sorted(error(rid, pos, rounded[rid][pos]) for rid, pos in got)
        median_most, mean_most = 3 * alone[n // 2], max(mean_most, 3 * sum(alone) / n)
        over_most = max(1, 0.02 * n + 3 * sum(e > tol for e in alone))
    print("%s: median %.3g (most %.3g) mean %.3g (most %.3g), %d of %d beyond %.3g" % (what, middle, median_most, sum(errs) / n, mean_most, over, n, tol))
    assert over <= over_most, "%s: %d of %d positions beyond %.3g" % (what, over, n, tol)
    assert middle <= median_most, "%s: median error %.3g (allowed %.3g)" % (what, middle, median_most)
    assert sum(errs) / n <= mean_most, "%s: mean error %.3g (allowed %.3g)" % (what, sum(errs) / n, mean_most)
    return errs[-1], None


def _dev(t):
    return t.cuda()


def _i32(v):
    return torch.tensor(list(v), dtype=torch.int32, device="cuda")


def _moe(experts, top, ff, limit, groups=None, identity=0, scale=1.0):
    r = {"experts": experts, "top": top, "scale": scale}
    if groups:
        r["groups"] = {"count": groups[0], "keep": groups[1]}
    if identity:
        r["identity"] = identity
    return {"kind": "moe", "router": r, "expert": {"ff": ff, "limit": limit}}


def _delta(heads, kv_heads, dim, vdim, conv, mlp):
    return {"type": "channel_delta", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}, "mlp": mlp}


def _gla(heads, dim, vdim, tau, mlp):
    return {"type": "gla", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau}, "mlp": mlp}


def _parallel(left, right, scales, mlp):
    """left: (heads, kv heads, dim, vdim, conv, scale, rotated entries, base); right: (heads, dim, vdim, cap)."""
    a = dict(zip(("heads", "kv_heads", "dim", "vdim", "conv", "scale"), left))
    if left[6]:
        a["rot"] = {"dims": left[6], "base": left[7]}
    b = dict(zip(("heads", "dim", "vdim", "gate_cap"), right))
    return {"type": "parallel", "mixer": {"left": a, "right": b, "left_scale": scales[0], "right_scale": scales[1]}, "mlp": mlp}


# K1: fewer query/key heads than heads in the delta rule, key and value sizes that differ everywhere, a part of every head
# rotated, gates with a low cap, twelve router outputs (three of them identity experts) in three groups of which two stay.
K1 = {"architecture": "Pekarax", "vocab": 211, "width": 96, "norm": {"eps": 1e-5}, "postln_alpha": 1.7,
      "layers": [_delta(4, 2, 24, 40, 4, _moe(9, 3, 48, 2.0, (3, 2), 3, 1.5)),
                 _parallel((4, 2, 32, 64, 3, 0.3, 16, 10000.0), (3, 20, 28, 4.0), (0.8, 1.3), _moe(4, 2, 40, 0.7, (2, 2), 0, 0.6)),
                 _gla(3, 20, 36, 4.0, _moe(6, 1, 32, 7.0, (4, 1), 2, 1.0))]}
# K2: sizes that are no multiple of 4 or 8, one tap (no convolution state), as many kv heads as heads, every entry of a head
# rotated, a layer without a feed-forward, one expert chosen of three in one group, a single head, constants of one, two
# parallel layers in a row.
K2 = {"architecture": "Pekarax", "vocab": 97, "width": 70, "norm": {"eps": 1e-6}, "postln_alpha": 1.0,
      "layers": [_parallel((3, 3, 10, 12, 1, 0.4, 10, 77.0), (1, 9, 11, 15.0), (1.0, 1.0), None),
                 _parallel((2, 1, 6, 14, 2, 1.0, 2, 500.0), (2, 5, 3, 30.0), (1.0, -0.5), _moe(3, 1, 30, 1.0)),
                 _gla(1, 7, 13, 1.0, None),
                 _delta(3, 3, 6, 9, 1, _moe(5, 3, 22, 3.0, None, 1, 2.5))]}
# K3: the tiled attention kernels' sizes (128 with three query heads a kv head), large head sizes in the recurrences, values
# shorter than keys, five taps, four experts of sixteen out of two groups of eight, a delta layer last and first.
K3 = {"architecture": "Pekarax", "vocab": 300, "width": 128, "norm": {"eps": 1e-5}, "postln_alpha": 4.0,
      "layers": [_delta(2, 1, 128, 64, 5, _moe(16, 4, 32, 2.0, (8, 2))),
                 _gla(2, 136, 72, 16.0, _moe(7, 2, 64, 1.2, (2, 1), 1, 2.0)),
                 _parallel((6, 2, 128, 64, 4, 0.25, 64, 300000.0), (2, 160, 96, 8.0), (1.1, 0.9), None),
                 _parallel((5, 5, 64, 64, 2, 0.125, 64, 1000.0), (4, 32, 16, 15.0), (0.5, 1.5), _moe(4, 4, 24, 1.5)),
                 _delta(6, 2, 32, 32, 2, None)]}
SHARP = dict(K1, norm={"eps": 1e-2})
CONFIGS = {"K1": K1, "K2": K2, "K3": K3}
LENGTHS = {"K1": [1, 2, 130, 61, 210, 37], "K2": [3, 75, 1, 140, 18, 66], "K3": [2, 90, 17, 1, 260, 40]}


def _write_model(folder, cfg, seed):
    from safetensors.torch import save_file
    os.makedirs(folder, exist_ok=True)
    W = P.random_weights(cfg, seed, ranks=(5 + seed % 9, 12 + seed % 7))
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file({k: v.to(torch.bfloat16).contiguous() for k, v in W.items()}, os.path.join(folder, "model.safetensors"))
    return W


_models, _engines, _plain = {}, {}, {}


def _model(tmp_path_factory, name):
    if name not in _models:
        folder = os.path.join(str(tmp_path_factory.getbasetemp()), "pekarax_" + name)
        _models[name] = (folder, _write_model(folder, CONFIGS[name], seed=len(name) + ord(name[-1])))
    return _models[name]


def _engine(tmp_path_factory, name, dtype, max_tokens, page_size=16, max_requests=4):
    from infinicore_infer_amd.engine import Engine
    key = (name, dtype, max_tokens, page_size, max_requests)
    if key not in _engines:
        folder, _ = _model(tmp_path_factory, name)
        _engines[key] = Engine.from_dir(folder, dtype=dtype, max_tokens=max_tokens, page_size=page_size, max_requests=max_requests)
    return _engines[key]


def _requests(name, seed=0):
    return {"r%d" % i: H.random_tokens(CONFIGS[name]["vocab"], n, seed * 100 + i) for i, n in enumerate(LENGTHS[name])}


def _reference(tmp_path_factory, name, requests):
    key = (name, tuple(sorted((k, tuple(v)) for k, v in requests.items())))
    if key not in _plain:
        _, W = _model(tmp_path_factory, name)
        _plain[key] = {rid: P.forward(CONFIGS[name], W, toks, torch.float64) for rid, toks in requests.items()}
    return _plain[key]


MODES = {
    "whole": H.trace_whole,
    "tail": lambda r: H.trace_last_one_by_one(r, tail=100),     # long decoding: states move on token by token
    "chunks": H.trace_chunks,
    "mixed": H.trace_mixed,
}


@pytest.mark.parametrize("mode", list(MODES))
@pytest.mark.parametrize("dname,dtype,tol", DTYPES)
@pytest.mark.parametrize("name", list(CONFIGS))
def test_replay_modes(tmp_path_factory, name, dname, dtype, tol, mode):
    """Prefill against token-by-token decoding, portions down to two tokens, unequal requests in one batch with pages
    and state slots used again: every position's logits against the plain implementation."""
    requests = _requests(name)
    steps, max_tokens = MODES[mode](requests)
    engine = _engine(tmp_path_factory, name, dtype, max_tokens)
    ref = _reference(tmp_path_factory, name, requests)
    got = H.run_trace(engine, steps)
    assert len(got) == sum(len(t) for t in requests.values())
    worst = _compare(got, ref, dtype, tol, "%s %s %s" % (name, dname, mode))
    print("worst error %.3g at %s (allowed %.3g)" % (worst[0], worst[1], tol))
    engine.cache.check_invariants()
    assert not engine.cache.requests
    for g in range(len(engine.groups)):
        assert engine.cache.free_pages(g) == engine.num_pages


# ---- the comparison is sharp enough -------------------------------------------------------------------------------------
def _with_weights(monkeypatch, change):
    """The plain implementation on changed weights: ``change(name, tensor)``."""
    real = P.forward
    monkeypatch.setattr(P, "forward", lambda cfg, W, tokens, dtype=torch.float64, layers_out=None: real(
        cfg, {k: change(k, v) for k, v in W.items()}, tokens, dtype, layers_out))


def _with_config(monkeypatch, change):
    real = P.forward

    def changed(cfg, W, tokens, dtype=torch.float64, layers_out=None):
        cfg = json.loads(json.dumps(cfg))
        change(cfg)
        return real(cfg, W, tokens, dtype, layers_out)
    monkeypatch.setattr(P, "forward", changed)


def _routed(monkeypatch, choose=None, weight=None, identity=True, scores=None):
    """The routed feed-forward with one piece replaced: who is chosen, what a chosen one weighs, the scores."""
    def routed(h, W, p, mlp):
        r = mlp["router"]
        groups = r.get("groups") or {"count": 1, "keep": 1}
        s = (scores or (lambda z, r: torch.softmax(z, -1)))(h @ W[p + "router"].T, r)
        out = torch.zeros_like(h)
        for t in range(h.shape[0]):
            chosen = (choose or P.choose)(s[t], W[p + "correction"], r["top"], groups["count"], groups["keep"])
            w = (weight or (lambda s, c, e, chosen, r: s[e] / (sum(s[x] for x in chosen) + 1e-20) * r["scale"]))
            for e in chosen:
                if e >= r["experts"]:
                    y = h[t] if identity else torch.zeros_like(h[t])
                else:
                    y = P.bounded_unit(h[t][None], W, "%se%d." % (p, e), mlp["expert"]["limit"])[0]
                out[t] = out[t] + w(s[t], W[p + "correction"], e, chosen, r) * y
        return out
    monkeypatch.setattr(P, "routed_experts", routed)


def _delta_memory(order):
    def memory(q, k, v, decay, beta):
        T, heads, dim = q.shape
        S = torch.zeros(heads, dim, v.shape[2], dtype=q.dtype)
        out = torch.zeros(T, heads, v.shape[2], dtype=q.dtype)
        read = lambda S, x: (S * x[:, :, None]).sum(1)
        for t in range(T):
            g = decay[t][:, :, None]
            if order == "read first":
                S = g * S
                out[t] = read(S, q[t])
                S = S + k[t][:, :, None] * (beta[t][:, None] * (v[t] - read(S, k[t])))[:, None, :]
            elif order == "error before the decay":
                u = beta[t][:, None] * (v[t] - read(S, k[t]))
                S = g * S + k[t][:, :, None] * u[:, None, :]
                out[t] = read(S, q[t])
            elif order == "decay last":
                S = g * (S + k[t][:, :, None] * (beta[t][:, None] * (v[t] - read(S, k[t])))[:, None, :])
                out[t] = read(S, q[t])
            else:                                           # no delta rule
                S = g * S + k[t][:, :, None] * (beta[t][:, None] * v[t])[:, None, :]
                out[t] = read(S, q[t])
        return out
    return memory


def _mlstm(floor=True, norm=True):
    def memory(q, k, v, log_i, log_f):
        T, heads, dim = q.shape
        S, n = torch.zeros(heads, dim, v.shape[2], dtype=q.dtype), torch.zeros(heads, dim, dtype=q.dtype)
        m = torch.zeros(heads, dtype=q.dtype)
        out = torch.zeros(T, heads, v.shape[2], dtype=q.dtype)
        for t in range(T):
            m_new = torch.maximum(log_f[t] + m, log_i[t])
            keep, add = torch.exp(log_f[t] + m - m_new), torch.exp(log_i[t] - m_new)
            S = keep[:, None, None] * S + add[:, None, None] * k[t][:, :, None] * v[t][:, None, :]
            n = keep[:, None] * n + add[:, None] * k[t]
            m = m_new
            nq = (n * q[t]).sum(-1).abs()
            den = (torch.maximum(nq, torch.exp(-m)) if floor else nq) + 1e-6 if norm else torch.ones_like(nq)
            out[t] = (S * q[t][:, :, None]).sum(1) / den[:, None]
        return out
    return memory


def _misread(monkeypatch, what):
    """One plausible misreading put into the plain implementation."""
    put = lambda name, f: monkeypatch.setattr(P, name, f)
    conv = P.short_conv
    if what == "the norm before the sublayers":
        put("sum_then_norm", lambda x, y, w, alpha, eps: alpha * x + y)
    elif what == "no alpha":
        put("sum_then_norm", lambda x, y, w, alpha, eps: P.unit_rms(x + y, eps) * (1.0 + w))
    elif what == "alpha on the result":
        put("sum_then_norm", lambda x, y, w, alpha, eps: P.unit_rms(x + alpha * y, eps) * (1.0 + w))
    elif what == "a norm's weight around one":
        put("sum_then_norm", lambda x, y, w, alpha, eps: P.unit_rms(alpha * x + y, eps) * w)
    elif what == "taps in reverse":
        put("short_conv", lambda x, w: conv(x, w.flip(1)))
    elif what == "the convolution sees one token less":
        put("short_conv", lambda x, w: conv(x, torch.cat([torch.zeros_like(w[:, :1]), w[:, 1:]], 1)))
    elif what == "adjacent pairs rotated":
        def pairs(x, positions, dims, base):
            order = [j for i in range(dims // 2) for j in (i, i + dims // 2)]
            y = x.clone()
            y[..., order] = x[..., :dims]                 # entry pairs (2i, 2i+1) where the halves' were
            z = real(torch.cat([x[..., 0:dims:2], x[..., 1:dims:2], x[..., dims:]], -1), positions, dims, base)
            out = x.clone()
            out[..., 0:dims:2], out[..., 1:dims:2] = z[..., :dims // 2], z[..., dims // 2:dims]
            return out
        real = P.rotate_halves
        put("rotate_halves", pairs)
    elif what == "positions from one":
        # a shift of all positions changes no score: shift the queries' alone
        real = P.rotate_halves
        put("rotate_halves", lambda x, positions, dims, base: real(x, [p + (x.shape[1] == 4) for p in positions], dims, base))
    elif what == "frequencies over the whole head":
        real = P.rotate_halves

        def whole(x, positions, dims, base):
            return real(x, positions, dims, base ** (dims / x.shape[-1]))
        put("rotate_halves", whole)
    elif what == "no norm on queries and keys":
        real = P.conv_attention

        def bare(h, W, p, *a):
            unit = P.unit_rms
            P.unit_rms = lambda x, eps: x
            try:
                return real(h, W, p, *a)
            finally:
                P.unit_rms = unit
        put("conv_attention", bare)
    elif what == "scores over the root of the size":
        _with_config(monkeypatch, lambda c: c["layers"][1]["mixer"]["left"].update(scale=c["layers"][1]["mixer"]["left"]["dim"] ** -0.5))
    elif what == "no scale on the left":
        _with_config(monkeypatch, lambda c: c["layers"][1]["mixer"].update(left_scale=1.0))
    elif what == "no scale on the right":
        _with_config(monkeypatch, lambda c: c["layers"][1]["mixer"].update(right_scale=1.0))
    elif what == "no floor under the denominator":
        put("matrix_memory", _mlstm(floor=False))
    elif what == "no denominator":
        put("matrix_memory", _mlstm(norm=False))
    elif what == "no cap on the gates":
        _with_config(monkeypatch, lambda c: c["layers"][1]["mixer"]["right"].update(gate_cap=1e9))
    elif what == "no input gate's bias":
        _with_weights(monkeypatch, lambda k, v: torch.zeros_like(v) if k.endswith(".i.b") else v)
    elif what == "no forget gate's bias":
        _with_weights(monkeypatch, lambda k, v: torch.zeros_like(v) if k.endswith(".f.b") else v)
    elif what == "tau left out":
        _with_config(monkeypatch, lambda c: c["layers"][2]["mixer"].update(tau=1.0))
    elif what == "no bias on the decay":
        _with_weights(monkeypatch, lambda k, v: torch.zeros_like(v) if k.endswith((".a2.b", ".dt_bias")) else v)
    elif what == "a sigmoid gate in linear attention":
        put("gla_mixer", _gla_with_sigmoid)
    elif what in ("read first", "error before the decay", "decay last", "no delta rule"):
        put("delta_memory", _delta_memory(what))
    elif what == "queries and keys not of unit length":
        put("unit_length", lambda x: x)
    elif what == "unit root mean square instead of unit length":
        put("unit_length", lambda x: P.unit_rms(x, 1e-6))
    elif what == "heads share query/key heads in turn":
        real = torch.Tensor.repeat_interleave
        monkeypatch.setattr(torch.Tensor, "repeat_interleave", lambda x, n, d: x.repeat(1, n, 1) if d == 1 else real(x, n, d))
    elif what == "decay rate not exponentiated":
        _with_weights(monkeypatch, lambda k, v: torch.log(v.abs() + 1e-9) if k.endswith(".A_log") else v)
    elif what == "weights with the correction":
        _routed(monkeypatch, weight=lambda s, c, e, chosen, r: (s + c)[e] / (sum((s + c)[x] for x in chosen) + 1e-20) * r["scale"])
    elif what == "choice without the correction":
        _routed(monkeypatch, choose=lambda s, c, top, n, keep: P.choose(s, torch.zeros_like(c), top, n, keep))
    elif what == "no groups":
        _routed(monkeypatch, choose=lambda s, c, top, n, keep: P.choose(s, c, top, 1, 1))
    elif what == "a group is as good as its sum":
        def by_sum(s, c, top, n, keep):
            a = [float(x) for x in s + c]
            size = len(a) // n
            kept = sorted(range(n), key=lambda g: -sum(a[g * size:(g + 1) * size]))[:keep]
            return sorted((e for e in range(len(a)) if e // size in kept), key=lambda e: -a[e])[:top]
        _routed(monkeypatch, choose=by_sum)
    elif what == "experts of other groups count as zero":
        def zeros(s, c, top, n, keep):
            a = [float(x) for x in s + c]
            size = len(a) // n
            kept = sorted(range(n), key=lambda g: -max(a[g * size:(g + 1) * size]))[:keep]
            a = [x if e // size in kept else 0.0 for e, x in enumerate(a)]
            return sorted(range(len(a)), key=lambda e: -a[e])[:top]
        _routed(monkeypatch, choose=zeros)
    elif what == "identity experts give nothing":
        _routed(monkeypatch, identity=False)
    elif what == "softmax without the identity experts":
        _routed(monkeypatch, scores=lambda z, r: torch.cat([torch.softmax(z[:, :r["experts"]], -1), torch.sigmoid(z[:, r["experts"]:])], -1))
    elif what == "weights not divided by their sum":
        _routed(monkeypatch, weight=lambda s, c, e, chosen, r: s[e] * r["scale"])
    elif what == "no scale on the weights":
        _routed(monkeypatch, weight=lambda s, c, e, chosen, r: s[e] / sum(s[x] for x in chosen))
    elif what == "the gate bounded on both sides":
        put("bounded_unit", _unit(lambda g, l: torch.clamp(g, -l, l)))
    elif what == "no one on the up branch":
        put("bounded_unit", _unit(one=0.0))
    elif what == "a plain silu in the experts":
        put("bounded_unit", _unit(slope=1.0))
    else:
        raise ValueError(what)


def _unit(bound=lambda g, l: torch.clamp(g, max=l), one=1.0, slope=1.702):
    def unit(h, W, p, limit):
        g, u = bound(h @ W[p + "gate"].T, limit), torch.clamp(h @ W[p + "up"].T, -limit, limit)
        return (g * torch.sigmoid(slope * g) * (u + one)) @ W[p + "down"].T
    return unit


def _gla_with_sigmoid(h, W, p, heads, dim, vdim, tau, eps):
    T = h.shape[0]
    q, k, v = ((h @ W[p + n].T).reshape(T, heads, -1) for n in ("q", "k", "v"))
    decay = torch.sigmoid((h @ W[p + "a1"].T) @ W[p + "a2"].T + W[p + "a2.b"]).pow(1 / tau).reshape(T, heads, dim)
    o = P.unit_rms(P.channel_decay_memory(q * dim ** -0.5, k, v, decay), eps) * W[p + "norm"]
    return (o.reshape(T, -1) * torch.sigmoid(h @ W[p + "g"].T)) @ W[p + "o"].T


MISREADINGS = [
    "the norm before the sublayers", "no alpha", "alpha on the result", "a norm's weight around one", "taps in reverse",
    "the convolution sees one token less", "adjacent pairs rotated", "positions from one", "frequencies over the whole head",
    "no norm on queries and keys", "scores over the root of the size", "no scale on the left", "no scale on the right",
    "no floor under the denominator", "no denominator", "no cap on the gates",
    "no input gate's bias", "no forget gate's bias", "tau left out", "no bias on the decay", "a sigmoid gate in linear attention",
    "read first", "error before the decay", "decay last", "no delta rule", "queries and keys not of unit length",
    "unit root mean square instead of unit length", "heads share query/key heads in turn", "decay rate not exponentiated",
    "weights with the correction", "choice without the correction", "no groups", "a group is as good as its sum",
    "experts of other groups count as zero", "identity experts give nothing", "softmax without the identity experts",
    "weights not divided by their sum", "no scale on the weights", "the gate bounded on both sides", "no one on the up branch",
    "a plain silu in the experts"]


@pytest.fixture(scope="module")
def sharp_run(tmp_path_factory):
    """One request through the float32 engine: the misreadings are held against its logits.  The correction is pulled down in
    every layer, so that choice scores are negative, and eps is large, so that the size of what a norm gets counts (the matrix
    memory's denominator is a factor per head and token, which a norm takes out again up to its eps; where the running maximum
    starts is seen in the gates alone, and tested there)."""
    from infinicore_infer_amd.engine import Engine
    from safetensors.torch import save_file
    folder = os.path.join(str(tmp_path_factory.getbasetemp()), "pekarax_sharp")
    os.makedirs(folder)
    W = P.random_weights(SHARP, 33)
    W = {k: ((v - 0.4).to(torch.bfloat16).float() if k.endswith(".correction") else v) for k, v in W.items()}
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(SHARP, f)
    save_file({k: v.to(torch.bfloat16).contiguous() for k, v in W.items()}, os.path.join(folder, "model.safetensors"))
    toks = H.random_tokens(K1["vocab"], 120, 21)
    engine = Engine.from_dir(folder, dtype=torch.float32, max_tokens=128, page_size=16, max_requests=1)
    steps, _ = H.trace_whole({"a": toks})
    got = H.run_trace(engine, steps)
    H.compare(got, {"a": P.forward(SHARP, W, toks, torch.float64)}, 2e-4, "as designed")
    return W, toks, got


@pytest.mark.parametrize("what", MISREADINGS)
def test_a_misreading_of_the_design_shows(sharp_run, monkeypatch, what):
    """The comparison the other tests rest on is sharp enough: with one misreading in the plain implementation the float32
    engine no longer agrees with it (the same request agrees without)."""
    W, toks, got = sharp_run
    _misread(monkeypatch, what)
    with pytest.raises(AssertionError):
        H.compare(got, {"a": P.forward(SHARP, W, toks, torch.float64)}, 2e-4, what)


def test_the_residual_stream_after_every_layer(tmp_path_factory):
    """Layer by layer in float32: the stream after every layer."""
    from infinicore_infer_amd.engine import Engine, StepEntry
    folder, W = _model(tmp_path_factory, "K3")
    toks = H.random_tokens(K3["vocab"], 45, 3)
    want = []
    P.forward(K3, W, toks, torch.float64, layers_out=want)
    eng = Engine.from_dir(folder, dtype=torch.float32, max_tokens=64, max_requests=1)
    got, build = [], eng._build_context

    def probed(entries, starts):
        ctx = build(entries, starts)
        ctx.layer_probe = lambda i, x, pending: got.append(x.clone())
        return ctx
    eng._build_context = probed
    eng.step([StepEntry("a", toks, [])])
    assert len(want) == 5 and len(got) >= 5
    for i, w in enumerate(want):
        assert torch.allclose(got[i].cpu().double(), w, atol=3e-5 * float(w.abs().max())), "after layer %d" % i


@pytest.mark.parametrize("name,page_size", [("K1", 64), ("K3", 32)])
def test_other_page_sizes(tmp_path_factory, name, page_size):
    requests = _requests(name, seed=2)
    steps, max_tokens = H.trace_mixed(requests, seed=5)
    ref = _reference(tmp_path_factory, name, requests)
    engine = _engine(tmp_path_factory, name, torch.float32, max_tokens + 4 * page_size, page_size=page_size)
    H.compare(H.run_trace(engine, steps), ref, 2e-4, "%s page %d" % (name, page_size))
    engine.cache.check_invariants()


@pytest.mark.parametrize("name", ["K1", "K3"])
def test_recorded_decode_steps_equal_eager_ones(tmp_path_factory, name):
    """Long decoding: the same request decoded through recorded steps and eagerly gives the same logits; states, running
    maxima and convolution inputs move on exactly once per step, also in the step that is recorded."""
    from infinicore_infer_amd.engine import Engine, StepEntry
    folder, W = _model(tmp_path_factory, name)
    cfg = CONFIGS[name]
    toks = H.random_tokens(cfg["vocab"], 200, 9)
    rows = {}
    for graphs in (True, False):
        eng = Engine.from_dir(folder, dtype=torch.float32, max_tokens=512, page_size=16, max_requests=2, use_graphs=graphs)
        eng.step([StepEntry("a", toks[:30], [])])
        out = []
        for t in toks[30:]:
            out.append(eng.step([StepEntry("a", [t], [0])]).float().cpu().clone())
        rows[graphs] = torch.cat(out)
        if graphs:
            assert eng.graph_replays > 100
    assert torch.equal(rows[True], rows[False])
    ref = P.forward(cfg, W, toks, torch.float64)[30:]
    assert float((rows[True].double() - ref).abs().max()) <= 2e-4 * float(ref.abs().max())


def test_a_forked_request_goes_on_apart(tmp_path_factory):
    """A copy of a request (its pages and its states) and the original continue with different tokens."""
    from infinicore_infer_amd.engine import Engine, StepEntry
    folder, W = _model(tmp_path_factory, "K1")
    toks = H.random_tokens(K1["vocab"], 70, 11)
    a_tail, b_tail = H.random_tokens(K1["vocab"], 30, 12), H.random_tokens(K1["vocab"], 30, 13)
    eng = Engine.from_dir(folder, dtype=torch.float32, max_tokens=512, page_size=16, max_requests=3, use_graphs=False)
    eng.step([StepEntry("a", toks, [])])
    eng.fork("a", "b")
    la = eng.step([StepEntry("a", a_tail, list(range(30)))]).float().cpu().clone()
    lb = eng.step([StepEntry("b", b_tail, list(range(30)))]).float().cpu().clone()
    for got, tail in ((la, a_tail), (lb, b_tail)):
        ref = P.forward(K1, W, toks + tail, torch.float64)[70:]
        assert float((got.double() - ref).abs().max()) <= 2e-4 * float(ref.abs().max())
    eng.free("a")
    eng.free("b")
    eng.cache.check_invariants()


# ---- each mechanism's kernel alone ----------------------------------------------------------------------------------------
LENS = [203, 40, 9]
# the requests' tokens cut into steps: whole portions, portions of two, single tokens beside portions, single tokens alone, a
# request left out of a step
STEPS = [[(0, 33), (1, 2), (2, 1)], [(1, 16), (0, 1)], [(2, 1), (0, 2), (1, 1)], [(0, 1), (1, 1), (2, 1)], [(1, 18)], [(2, 4), (0, 17)],
         [(0, 1), (2, 1)], [(0, 146), (1, 1)], [(1, 1), (0, 2), (2, 1)]]
SLOTS = [4, 1, 2]                                                  # of five; the others hold NaN


def _walk(steps=STEPS):
    """Per step: (token rows as (request, position), token_req, request starts, slots, single)."""
    at = [0] * len(LENS)
    for step in steps:
        rows, req, starts = [], [], [0]
        for i, (r, n) in enumerate(step):
            rows += [(r, at[r] + j) for j in range(n)]
            req += [i] * n
            starts.append(starts[-1] + n)
            at[r] += n
        yield rows, _i32(req), _i32(starts), _i32([SLOTS[r] for r, _ in step]), all(n == 1 for _, n in step)
    assert at == LENS


def _pick(per_request, rows):
    return torch.stack([per_request[r][p] for r, p in rows])


def _fresh_state(size, pad=8):
    """A state row per slot: zeros in the slots in use, NaN in the others and in front of the state."""
    st = torch.full((5, pad + size), float("nan"), device="cuda")
    for s in SLOTS:
        st[s, pad:] = 0.0
    return st, pad


def _close(got, want, tol, what):
    err = float((got.float().cpu().double() - want).abs().max()) / max(1e-6, float(want.abs().max()))
    assert math.isfinite(err) and err <= tol, "%s: error %.3g (allowed %.3g)" % (what, err, tol)


MEMORY_SIZES = [  # heads, query/key heads, key size, value size
    (4, 2, 24, 40), (3, 3, 6, 9), (2, 1, 128, 64), (1, 1, 200, 33), (2, 1, 300, 24), (1, 1, 600, 20), (5, 5, 32, 32), (8, 4, 64, 128)]


@pytest.mark.parametrize("columns", [1, 2])
@pytest.mark.parametrize("H_,G,dk,dv", MEMORY_SIZES)
def test_delta_rule_over_portions_and_single_tokens(H_, G, dk, dv, columns):
    """The recurrence with a decay per key channel: slow decays (some exactly one), so that early writes still count at the
    end; the last query of every request is the first token's key."""
    from infinicore_infer_amd.kernels import ops
    g = torch.Generator().manual_seed(dk + dv)
    q, k = ([P.unit_length(torch.randn(n, G, dk, generator=g)) for n in LENS] for _ in range(2))
    for r in range(len(LENS)):
        q[r][-1] = k[r][0]
    v = [torch.randn(n, H_, dv, generator=g) for n in LENS]
    decay = [torch.exp(-0.2 * torch.rand(n, H_, dk, generator=g) * (torch.rand(n, H_, dk, generator=g) < 0.5)) for n in LENS]
    beta = [torch.sigmoid(torch.randn(n, H_, generator=g)) for n in LENS]
    rep = lambda x: x.double().repeat_interleave(H_ // G, 1)
    want = [P.delta_memory(rep(q[r]) * dk ** -0.5, rep(k[r]), v[r].double(), decay[r].double(), beta[r].double()) for r in range(len(LENS))]
    st, pad = _fresh_state(H_ * dv * dk)
    for rows, req, starts, slots, single in _walk():
        T = len(rows)
        qkv = torch.cat([_pick(q, rows).view(T, -1), _pick(k, rows).view(T, -1), _pick(v, rows).view(T, -1)], 1).cuda()
        nq = G * dk
        out = torch.full((T, H_ * dv), float("nan"), device="cuda")
        ops.matrix_memory(qkv[:, :nq], qkv[:, nq:2 * nq], qkv[:, 2 * nq:], _pick(decay, rows).view(T, -1).cuda(), H_, G, dk, dv, out, st, pad,
                          starts, slots, len(slots), single, scale=_pick(beta, rows).cuda(), delta=True, q_scale=dk ** -0.5,
                          columns_a_thread=columns)
        _close(out, _pick(want, rows).view(T, -1), 2e-5, "rows %s.." % (rows[0],))
    assert torch.isnan(st[0]).all() and torch.isnan(st[3]).all() and torch.isnan(st[:, :pad]).all()


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("columns", [1, 2])
@pytest.mark.parametrize("H_,G,dk,dv", MEMORY_SIZES)
def test_linear_attention_with_a_decay_per_channel(H_, G, dk, dv, columns, dtype):
    from infinicore_infer_amd.kernels import ops
    g = torch.Generator().manual_seed(dk + dv)
    q, k = ([torch.randn(n, G, dk, generator=g).to(dtype) for n in LENS] for _ in range(2))
    for r in range(len(LENS)):
        q[r][-1] = 3 * k[r][0]
    v = [torch.randn(n, H_, dv, generator=g).to(dtype) for n in LENS]
    decay = [torch.exp(-0.3 * torch.rand(n, H_, dk, generator=g) * (torch.rand(n, H_, dk, generator=g) < 0.7)) for n in LENS]
    rep = lambda x: x.double().repeat_interleave(H_ // G, 1)
    want = [P.channel_decay_memory(rep(q[r]) * 0.5, rep(k[r]), v[r].double(), decay[r].double()) for r in range(len(LENS))]
    st, pad = _fresh_state(H_ * dv * dk)
    for rows, req, starts, slots, single in _walk():
        T, nq = len(rows), G * dk
        wide = torch.cat([_pick(q, rows).view(T, -1), _pick(k, rows).view(T, -1), _pick(v, rows).view(T, -1), torch.zeros(T, 3).to(dtype)], 1).cuda()
        out = torch.full((T, H_ * dv), float("nan"), device="cuda")
        ops.matrix_memory(wide[:, :nq], wide[:, nq:2 * nq], wide[:, 2 * nq:2 * nq + H_ * dv], _pick(decay, rows).view(T, -1).cuda(), H_, G, dk,
                          dv, out, st, pad, starts, slots, len(slots), single, q_scale=0.5, columns_a_thread=columns)
        _close(out, _pick(want, rows).view(T, -1), 2e-5, "rows %s.." % (rows[0],))


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H_,G,dk,dv", [s for s in MEMORY_SIZES if s[0] == s[1]] + [(2, 2, 128, 96), (3, 3, 256, 16)])
def test_matrix_memory_with_exponential_gates(H_, G, dk, dv, dtype):
    """Gates, recurrence, denominator, norm and output gate together: the running maximum, the keys' sum and the memory are
    carried over the steps; strong and weak gates, so that the floor under the denominator and the maximum both matter."""
    from infinicore_infer_amd.kernels import ops
    g = torch.Generator().manual_seed(dk + dv)
    cap, eps = 6.0, 0.05                                       # (a large eps: the denominator counts)
    q, k = ([torch.randn(n, H_, dk, generator=g).to(dtype) for n in LENS] for _ in range(2))
    v = [torch.randn(n, H_, dv, generator=g).to(dtype) for n in LENS]
    z = [torch.randn(n, 2 * H_, generator=g) * 4 for n in LENS]
    og = [torch.randn(n, H_ * dv, generator=g).to(dtype) for n in LENS]
    bi, bf, w = torch.randn(H_, generator=g), torch.randn(H_, generator=g) + 2, 1 + 0.3 * torch.randn(H_ * dv, generator=g)
    want = []
    for r in range(len(LENS)):
        zz = z[r].double()
        li = cap * torch.tanh((zz[:, :H_] + bi) / cap)
        lf = -P.softplus(-cap * torch.tanh((zz[:, H_:] + bf) / cap))
        o = P.matrix_memory(q[r].double() * dk ** -0.5, k[r].double(), v[r].double(), li, lf)
        want.append(P.unit_rms(o, eps).reshape(LENS[r], -1) * w * torch.sigmoid(og[r].double()))
    top = H_ * (dv + 1) * dk
    st, pad = _fresh_state(top + H_)
    n_small = 0
    for rows, req, starts, slots, single in _walk():
        T, nq = len(rows), H_ * dk
        wide = torch.cat([_pick(x, rows).view(T, -1) for x in (q, k, v, og)], 1).cuda()
        keep, add, floor, num = (torch.full((T, H_), float("nan"), device="cuda") for _ in range(4))
        ops.memory_gates(_pick(z, rows).cuda(), bi.cuda(), bf.cuda(), cap, keep, add, floor, st, pad + top, starts, slots, len(slots))
        o = torch.full((T, H_ * dv), float("nan"), device="cuda")
        ops.matrix_memory(wide[:, :nq], wide[:, nq:2 * nq], wide[:, 2 * nq:2 * nq + H_ * dv], keep, H_, H_, dk, dv, o, st, pad, starts, slots,
                          len(slots), single, scale=add, q_scale=dk ** -0.5, extra_out=num)
        n_small += int((num.abs() < floor).sum())
        out = torch.empty(T, H_ * dv, dtype=dtype, device="cuda")
        ops.gated_head_norm(o, wide[:, 2 * nq + H_ * dv:], w.cuda(), H_, eps, out, num=num, floor=floor)
        _close(out, _pick(want, rows).view(T, -1), 1e-4 if dtype == torch.float32 else 1e-2, "rows %s.." % (rows[0],))
    assert n_small > 0


@pytest.mark.parametrize("H_", [1, 3, 70])
def test_exponential_gates_over_long_portions(H_):
    """More tokens than a wave and than a block takes at a time, cut at places inside and at the borders of its runs; the running maximum
    starts at zero, falls slowly and is overtaken by single strong input gates."""
    from infinicore_infer_amd.kernels import ops
    T, cap = 2600, 9.0
    g = torch.Generator().manual_seed(H_)
    z = torch.cat([torch.randn(T, H_, generator=g) * 2 - 4, torch.randn(T, H_, generator=g) * 2 + 3], 1)
    z[300, :H_] = z[1800, :H_] = 12.0
    bi, bf = torch.randn(H_, generator=g), torch.randn(H_, generator=g)
    li = cap * torch.tanh((z[:, :H_].double() + bi) / cap)
    lf = -P.softplus(-cap * torch.tanh((z[:, H_:].double() + bf) / cap))
    m, keep, add, floor = torch.zeros(H_, dtype=torch.float64), [], [], []
    for t in range(T):
        new = torch.maximum(lf[t] + m, li[t])
        keep.append(torch.exp(lf[t] + m - new))
        add.append(torch.exp(li[t] - new))
        floor.append(torch.exp(-new))
        m = new
    for cuts in ([0, 2600], [0, 64, 128, 129, 131, 200, 511, 1535, 2600], [0, 1, 2, 65, 2113, 2600]):
        st = torch.zeros(1, H_ + 3, device="cuda")
        outs = [torch.empty(T, H_, device="cuda") for _ in range(3)]
        for a, b in zip(cuts, cuts[1:]):
            ops.memory_gates(z[a:b].contiguous().cuda(), bi.cuda(), bf.cuda(), cap, *[o[a:b] for o in outs], st, 3, _i32([0, b - a]), _i32([0]), 1)
        for o, want in zip(outs, (keep, add, floor)):
            assert torch.allclose(o.cpu().double(), torch.stack(want), rtol=5e-5, atol=1e-7)
        assert torch.allclose(st[0, 3:].cpu().double(), m, atol=5e-5)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H_,G,dk,dv,taps", [(4, 2, 24, 40, 4), (3, 3, 6, 9, 1), (2, 1, 128, 64, 5), (1, 1, 600, 300, 3), (6, 2, 32, 32, 2), (2, 2, 16, 8, 8)])
def test_rows_of_the_delta_rule(dtype, H_, G, dk, dv, taps):
    """Convolution, silu, unit length and step sizes; the convolution's inputs are carried over portions shorter and longer
    than its taps."""
    from infinicore_infer_amd.kernels import ops
    g = torch.Generator().manual_seed(dk + taps)
    C = 2 * G * dk + H_ * dv
    x = [(2 * torch.randn(n, C + H_ + 5, generator=g)).to(dtype) for n in LENS]
    w = torch.randn(C, taps, generator=g) / math.sqrt(taps)
    want, beta_want = [], []
    for r in range(len(LENS)):
        y = P.silu(P.short_conv(x[r][:, :C].double(), w.double()))
        qk = P.unit_length(y[:, :2 * G * dk].view(-1, 2 * G, dk)).reshape(LENS[r], -1)
        want.append(torch.cat([qk, y[:, 2 * G * dk:]], 1))
        beta_want.append(torch.sigmoid(x[r][:, C:C + H_].double()))
    st, pad = _fresh_state((taps - 1) * C)
    for rows, req, starts, slots, single in _walk():
        xx = _pick(x, rows).cuda()
        T = len(rows)
        out, beta = torch.full((T, C), float("nan"), device="cuda"), torch.full((T, H_), float("nan"), device="cuda")
        ops.delta_prep(xx[:, :C], w.cuda(), xx[:, C:C + H_], out, beta, G, H_, dk, dv, 1e-6, st, pad, req, starts, slots, len(slots), single)
        _close(out, _pick(want, rows), 1e-5, "rows %s.." % (rows[0],))
        assert torch.allclose(beta.cpu().double(), _pick(beta_want, rows), atol=1e-6)
    for r in range(len(LENS)):
        for j in range(taps - 1):
            assert torch.equal(st[SLOTS[r], pad + j * C:pad + (j + 1) * C].cpu(), x[r][LENS[r] - (taps - 1) + j, :C].float())


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("Hq,G,dk,dv,taps,rot,base,weights", [
    (4, 2, 32, 64, 3, 16, 10000.0, False), (3, 3, 10, 12, 1, 10, 77.0, False), (6, 2, 128, 64, 4, 64, 300000.0, True), (2, 1, 200, 40, 2, 0, None, False),
    (2, 2, 512, 512, 5, 512, 1e6, False), (4, 1, 64, 128, 0, 64, 500.0, True), (9, 3, 64, 32, 8, 2, 10.0, False), (32, 8, 128, 128, 4, 128, 5e5, False)])
def test_convolution_rotation_and_norm_with_the_cache_write(dtype, Hq, G, dk, dv, taps, rot, base, weights):
    """q, k and v through a convolution (its inputs carried over the steps), q and k turned in halves at the requests' positions
    (up to 60,000) and brought to unit root mean square; keys and values land in their pages."""
    from infinicore_infer_amd.kernels import ops
    from infinicore_infer_amd.parts.rotary import pair_frequencies
    page, eps = 16, 1e-5
    g = torch.Generator().manual_seed(dk + rot)
    C = (Hq + G) * dk + G * dv
    first = [0, 59900, 1000]
    x = [(2 * torch.randn(n, C + 8, generator=g)).to(dtype) for n in LENS]
    cw = torch.randn(C, taps, generator=g) / math.sqrt(taps) if taps else None
    qw, kw = (1 + 0.2 * torch.randn(dk, generator=g), 1 + 0.2 * torch.randn(dk, generator=g)) if weights else (None, None)
    want = []
    for r in range(len(LENS)):
        y = x[r][:, :C].double()
        if taps:
            y = P.short_conv(y, cw.double())
        q, k, v = y[:, :Hq * dk].view(-1, Hq, dk), y[:, Hq * dk:(Hq + G) * dk].view(-1, G, dk), y[:, (Hq + G) * dk:].view(-1, G, dv)
        pos = range(first[r], first[r] + LENS[r])
        if rot:
            q, k = P.rotate_halves(q, pos, rot, base), P.rotate_halves(k, pos, rot, base)
        q, k = P.unit_rms(q, eps), P.unit_rms(k, eps)
        want.append((q * (qw if weights else 1.0), k * (kw if weights else 1.0), v))
    freq = pair_frequencies(rot, base).cuda() if rot else None
    st, pad = _fresh_state(max(0, taps - 1) * C)
    kc = torch.zeros(10, G, page, dk, dtype=dtype, device="cuda")
    vc = torch.zeros(10, G, page, dv, dtype=dtype, device="cuda")
    tol = 2e-5 if dtype == torch.float32 else 3e-2
    rng = random.Random(3)
    for rows, req, starts, slots, single in _walk():
        T = len(rows)
        xx = _pick(x, rows).cuda()
        q_out = torch.full((T, Hq * dk), float("nan"), device="cuda").to(dtype)
        places = rng.sample(range(10 * page), T)
        ops.conv_rope_norm_store(xx, cw.cuda() if taps else None, _i32(first[r] + p for r, p in rows), freq, rot, qw.cuda() if weights else None,
                                 kw.cuda() if weights else None, True, eps, q_out, kc, vc, _i32(places), Hq, G, dk, dv, page,
                                 st if taps else None, pad, req, starts, slots, len(slots), single)
        kcpu, vcpu = kc.float().cpu().double(), vc.float().cpu().double()
        wq, wk, wv = ([want[r][i][p] for r, p in rows] for i in range(3))
        assert torch.allclose(q_out.float().cpu().double(), torch.stack(wq).view(T, -1), atol=tol * 4, rtol=tol)
        for t, s in enumerate(places):
            assert torch.allclose(kcpu[s // page, :, s % page], wk[t], atol=tol * 4, rtol=tol)
            assert torch.allclose(vcpu[s // page, :, s % page], wv[t], atol=tol * 4, rtol=tol)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("M,N,K,heads", [(1, 96, 5, 4), (7, 70, 12, 7), (65, 128, 24, 2), (200, 512, 64, 4), (130, 33, 16, 3)])
def test_decay_factors_from_a_low_rank_product(dtype, M, N, K, heads):
    from infinicore_infer_amd.kernels import ops
    g = torch.Generator().manual_seed(N + K)
    wide = torch.randn(M, K + 11, generator=g).to(dtype)
    a, w = wide[:, 3:3 + K], (2 * torch.randn(N, K, generator=g) / math.sqrt(K)).to(dtype)
    bias, rate = torch.randn(N, generator=g), torch.exp(torch.randn(heads, generator=g))
    z = a.double() @ w.double().T + bias
    out = torch.empty(M, N, device="cuda")
    ops.decay_product(wide.cuda()[:, 3:3 + K], w.cuda(), out, bias.cuda(), rate=rate.cuda())
    want = torch.exp(-rate.double().repeat_interleave(N // heads) * P.softplus(z))
    assert torch.allclose(out.cpu().double(), want, atol=3e-6)
    ops.decay_product(wide.cuda()[:, 3:3 + K], w.cuda(), out, bias.cuda(), log_scale=1 / 16.0)
    assert torch.allclose(out.cpu().double(), torch.sigmoid(z).pow(1 / 16.0), atol=3e-6)
    # the factors alone, from products that are there already, with arguments far out on both sides
    zf = (z * 12).float()
    z2 = zf.clone().cuda()
    ops.decay_rows(z2, bias.cuda(), rate=rate.cuda())
    assert torch.allclose(z2.cpu().double(), torch.exp(-rate.double().repeat_interleave(N // heads) * P.softplus(zf.double() + bias)), atol=3e-6)
    z2 = zf.clone().cuda()
    ops.decay_rows(z2, bias.cuda(), log_scale=0.25)
    assert torch.allclose(z2.cpu().double(), torch.sigmoid(zf.double() + bias).pow(0.25), atol=3e-6, rtol=1e-5)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("T,heads,dv,shared,gate,den", [(5, 3, 40, True, "silu", False), (9, 2, 9, False, "sigmoid", True), (3, 4, 300, True, "sigmoid", False),
                                                        (70, 8, 128, False, "silu", True), (2, 1, 1000, False, "sigmoid", True)])
def test_norm_per_head_under_a_gate(dtype, T, heads, dv, shared, gate, den):
    from infinicore_infer_amd.kernels import ops
    g = torch.Generator().manual_seed(dv)
    n, eps = heads * dv, 1e-4
    y, z = 0.1 * torch.randn(T, n, generator=g), (2 * torch.randn(T, n + 7, generator=g)).to(dtype)
    w = 1 + 0.3 * torch.randn(dv if shared else n, generator=g)
    num, floor = torch.randn(T, heads, generator=g), torch.exp(torch.randn(T, heads, generator=g))
    out = torch.empty(T, n, dtype=dtype, device="cuda")
    ops.gated_head_norm(y.cuda(), z.cuda()[:, 3:3 + n], w.cuda(), heads, eps, out, gate=gate, num=num.cuda() if den else None, floor=floor.cuda() if den else None)
    v = y.double().view(T, heads, dv)
    if den:
        v = v / (torch.maximum(num.double().abs(), floor.double()) + 1e-6)[:, :, None]
    zz = z[:, 3:3 + n].double()
    v = P.unit_rms(v, eps) * (w.double() if shared else w.double().view(heads, dv))
    want = v.reshape(T, n) * (torch.sigmoid(zz) if gate == "sigmoid" else P.silu(zz))
    _close(out, want, 2e-6 if dtype == torch.float32 else 5e-3, "norm per head")


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("T,d", [(5, 70), (3, 256), (2, 2304), (1, 8200), (130, 96)])
def test_norm_on_the_sum(dtype, T, d):
    from infinicore_infer_amd.kernels import ops
    g = torch.Generator().manual_seed(d)
    ya, yb = (torch.randn(T, d, generator=g).to(dtype) for _ in range(2))
    x, w, eps, alpha = torch.randn(T, d, generator=g), 1 + 0.3 * torch.randn(d, generator=g), 1e-5, 2.5
    for branches in (((ya, 1.0),), ((ya, 0.7), (yb, -1.4))):
        xs, copy = x.clone().cuda(), torch.empty(T, d, dtype=dtype, device="cuda")
        ops.sum_norm(tuple((y.cuda(), s) for y, s in branches), alpha, w.cuda(), xs, eps, copy=copy)
        want = P.sum_then_norm(x.double(), sum(s * y.double() for y, s in branches), w.double() - 1.0, alpha, eps)
        assert torch.allclose(xs.cpu().double(), want, atol=1e-5)
        assert torch.allclose(copy.float().cpu().double(), want, atol=1e-5 if dtype == torch.float32 else 3e-2)


@pytest.mark.parametrize("T,E,top,groups,keep,shift", [(40, 12, 3, 3, 2, 0.0), (40, 12, 3, 3, 2, -0.6), (7, 10, 2, 2, 1, 0.0), (33, 6, 6, 1, 1, 0.0),
                                                       (9, 150, 8, 10, 3, -0.1), (5, 1000, 16, 50, 2, 0.0), (20, 8, 1, 8, 1, -2.0), (6, 260, 5, 1, 1, 0.1)])
def test_choice_with_a_correction_and_in_groups(T, E, top, groups, keep, shift):
    """The choice goes by corrected scores (negative ones too: those of groups that fell out cannot be chosen, whatever the
    others are), the weights by the scores alone."""
    from infinicore_infer_amd.kernels import ops
    g = torch.Generator().manual_seed(E + T)
    z, corr = 2 * torch.randn(T, E, generator=g), 0.2 * torch.randn(E, generator=g) + shift
    z[0], z[1] = 0.5, z[1, 0]                              # ties broken by the correction alone
    ids = torch.empty(T, top, dtype=torch.int32, device="cuda")
    w = torch.empty(T, top, dtype=torch.float32, device="cuda")
    ops.moe_route(z.cuda(), top, ids, w, "softmax", True, corr.cuda(), groups, keep, 2.5)
    s = torch.softmax(z.double(), -1)
    want = [P.choose(s[t].float(), corr, top, groups, keep) for t in range(T)]
    assert ids.cpu().tolist() == want
    ws = torch.stack([s[t, want[t]] for t in range(T)])
    assert torch.allclose(w.cpu().double(), ws / ws.sum(-1, keepdim=True) * 2.5, atol=1e-5)
    # equal corrected scores: the lower index, of groups too
    ops.moe_route(torch.zeros(T, E, device="cuda"), top, ids, w, "softmax", True, torch.full((E,), -0.25, device="cuda"), groups, keep, 1.0)
    assert ids.cpu().tolist() == [list(range(top))] * T


@pytest.mark.parametrize("d,ff", [(48, 40), (64, 32), (70, 22)])
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_routed_experts_part_for_few_and_many_rows(dtype, d, ff):
    """The part with few rows (no integer leaves the device) and with many (one library product per expert) against the plain
    feed-forward: bounded units, weights on the output, identity experts, groups.  One batch chooses identity experts alone."""
    from infinicore_infer_amd.engine.context import StepContext, Workspace
    from infinicore_infer_amd.parts import Runtime
    from infinicore_infer_amd.parts.routed_experts import RoutedExperts
    mlp = _moe(6, 3, ff, 0.9, (4, 2), 2, 1.7)
    cfg = {"vocab": 8, "width": d, "layers": [_gla(1, 8, 8, 1.0, mlp)]}
    W = {k[len("l0.mlp."):]: v for k, v in P.random_weights(cfg, 5).items() if k.startswith("l0.mlp.")}
    ctx = StepContext()
    ctx.ws, ctx.cu_count = Workspace("cuda"), 256
    g = torch.Generator().manual_seed(3)
    for only_identity in (False, True):
        if only_identity:                                  # two of eight in one group of two: the identity experts' group
            mlp = _moe(6, 2, ff, 0.9, (4, 1), 2, 1.7)
            W = dict(W, correction=torch.tensor([0.0] * 6 + [3.0, 3.0]))
        r = mlp["router"]
        part = RoutedExperts("", Runtime(dtype, "cuda"), d, 6, r["top"], ff, None, scores="softmax", renormalize=True, weight_on="output",
                             correction=True, groups=4, group_keep=r["groups"]["keep"], identity=2, scale=1.7, unit="clamped", limit=0.9, slope=1.702)
        part.load_weights({k: (v if k == "correction" else v.to(dtype)).cuda() for k, v in W.items()})
        for T in (1, 7, 64, 65, 300):
            h = torch.randn(T, d, generator=g).to(dtype)
            got = part.forward(h.cuda(), ctx).float().cpu().double()
            want = P.routed_experts(h.double(), {k: v.double() for k, v in W.items()}, "", mlp)
            if only_identity:
                assert torch.allclose(want, 1.7 * h.double(), atol=1e-9)
            if dtype == torch.float32:
                assert torch.allclose(got, want, atol=2e-5 * float(want.abs().max())), T
            else:
                err = (got - want).abs().amax(-1) / float(want.abs().max())
                assert float(err.mean()) < 1e-2 and int((err > 5e-2).sum()) <= max(1, T // 30), (T, float(err.max()))


def test_mixers_side_by_side_without_a_block_that_sums(tmp_path_factory):
    """The part's own sum of its branches equals what the block's kernel makes of them."""
    from infinicore_infer_amd.engine import Engine, StepEntry
    folder, W = _model(tmp_path_factory, "K2")
    toks = H.random_tokens(K2["vocab"], 50, 8)
    eng = Engine.from_dir(folder, dtype=torch.float32, max_tokens=64, max_requests=1, use_graphs=False)
    for l in eng.model.layers:
        l.mixer.yields_branches = False
    got = eng.step([StepEntry("a", toks, list(range(50)))]).cpu().double()
    ref = P.forward(K2, W, toks, torch.float64)
    assert float((got - ref).abs().max()) <= 2e-4 * float(ref.abs().max())


# ---- generation through the entry point --------------------------------------------------------------------------------
def _plain_greedy(cfg, W, prompt, n):
    toks = list(prompt)
    for _ in range(n):
        toks.append(int(P.forward(cfg, W, toks, torch.float64)[-1].argmax()))
    return toks[len(prompt):]


@pytest.mark.parametrize("name", ["K1", "K2", "K3"])
def test_greedy_generation_through_the_entry_point_and_scheduler(tmp_path_factory, name):
    """Several prompts of unequal length through CausalLM.generate_batch (the scheduler: chunked prompts, continuous
    batching, recorded decode steps) in float32: the plain implementation's tokens."""
    from infinicore_infer_amd.causal_lm import CausalLM
    folder, W = _model(tmp_path_factory, name)
    cfg = CONFIGS[name]
    prompts = [H.random_tokens(cfg["vocab"], n, 40 + i) for i, n in enumerate([50, 3, 21])]
    model = CausalLM(folder, max_tokens=256, dtype=torch.float32, cache_tokens=1024, page_size=16, max_requests=4)
    outs = model.generate_batch(prompts, 10, max_batch_tokens=24, chunk_size=16)
    for p, o in zip(prompts, outs):
        assert o == _plain_greedy(cfg, W, p, 10)
    model.engine.cache.check_invariants()


def test_command_line_runs_the_design(tmp_path_factory):
    import subprocess
    import sys
    folder, W = _model(tmp_path_factory, "K2")
    prompt = H.random_tokens(K2["vocab"], 9, 77)
    r = subprocess.run([sys.executable, "-m", "infinicore_infer_amd.pekarax", "--amd", folder, "--dtype", "float32",
                        "--prompt-ids", ",".join(map(str, prompt)), "--max-new-tokens", "6", "--max-tokens", "128"],
                       cwd=H.__file__.rsplit("/tests/", 1)[0], capture_output=True, text=True, timeout=300)
    assert r.returncode == 0, r.stderr[-2000:]
    want = _plain_greedy(K2, W, prompt, 6)
    assert " ".join(map(str, want)) in " ".join(r.stdout.split()), r.stdout[-2000:]


def test_command_line_with_random_weights(tmp_path):
    import subprocess
    import sys
    path = str(tmp_path / "config.json")
    with open(path, "w") as f:
        json.dump(K3, f)
    r = subprocess.run([sys.executable, "-m", "infinicore_infer_amd.causal_lm", "--amd", "--random-weights", "--config", path,
                        "--prompt-len", "40", "--num-prompts", "3", "--max-new-tokens", "5", "--max-tokens", "256",
                        "--max-batch-tokens", "64", "--chunk-size", "32", "--weights-norm-std", "0.05"],
                       cwd=H.__file__.rsplit("/tests/", 1)[0], capture_output=True, text=True, timeout=300)
    assert r.returncode == 0, r.stderr[-2000:]
    assert r.stdout.count("tokens[") == 3, r.stdout[-2000:]


def test_trace_runner_as_a_program(tmp_path_factory, tmp_path):
    """bin/trace_run on a model folder: steps on standard input, logits files and 'done' lines out; a request left out of
    a step goes on later; pages and the state slots are used again."""
    import subprocess
    folder, W = _model(tmp_path_factory, "K2")
    requests = _requests("K2", seed=4)
    steps, max_tokens = H.trace_mixed(requests, seed=3)
    root = H.__file__.rsplit("/tests/", 1)[0]
    out = str(tmp_path / "out")
    r = subprocess.run([os.path.join(root, "bin", "trace_run"), "--model", folder, "--dtype", "float32", "--out", out,
                        "--max-tokens", str(max_tokens)], input="\n".join(json.dumps(s) for s in steps) + "\n",
                       capture_output=True, text=True, timeout=300, cwd=root)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [l for l in r.stdout.split("\n") if l.startswith("done")] == ["done %d" % s["step"] for s in steps]
    ref = {rid: P.forward(K2, W, toks, torch.float64) for rid, toks in requests.items()}
    at, got = {}, {}
    for s in steps:
        rows = torch.frombuffer(bytearray(open(os.path.join(out, "%d.f32" % s["step"]), "rb").read()), dtype=torch.float32).view(-1, K2["vocab"])
        i = 0
        for e in s["entries"]:
            for w in e["want"]:
                got[(e["id"], at.get(e["id"], 0) + w)] = rows[i].clone()
                i += 1
            at[e["id"]] = at.get(e["id"], 0) + len(e["tokens"])
        assert i == rows.shape[0]
    H.compare(got, ref, 2e-4, "trace runner", steps)


# ---- configurations drawn from seeds -------------------------------------------------------------------------------------
def _drawn_config(seed):
    rng = random.Random(seed)
    width = rng.choice([34, 48, 64, 100])

    def mlp():
        if rng.random() < 0.2:
            return None
        identity = rng.choice([0, 0, 1, 2, 5])
        experts = rng.choice([2, 3, 7, 11])
        total = experts + identity
        count = rng.choice([g for g in (1, 1, 2, 3, 4, 6) if total % g == 0])
        keep = rng.randint(1, count)
        top = rng.randint(1, min(4, keep * (total // count)))
        return _moe(experts, top, rng.choice([12, 30, 64]), round(rng.uniform(0.3, 3.0), 2), (count, keep) if rng.random() < 0.8 or count > 1 else None,
                    identity, round(rng.uniform(0.5, 3.0), 2))
    layers = []
    for _ in range(rng.choice([2, 3, 4])):
        kind = rng.choice(["channel_delta", "gla", "parallel"])
        if kind == "channel_delta":
            kv = rng.choice([1, 2, 3])
            layers.append(_delta(kv * rng.choice([1, 2, 3]), kv, rng.choice([4, 12, 32, 50]), rng.choice([5, 16, 33, 64]), rng.choice([1, 2, 3, 4, 6]), mlp()))
        elif kind == "gla":
            layers.append(_gla(rng.choice([1, 2, 3]), rng.choice([4, 12, 32, 70]), rng.choice([5, 16, 33, 64]), rng.choice([1.0, 4.0, 16.0]), mlp()))
        else:
            kv, dim = rng.choice([1, 2, 3]), rng.choice([8, 12, 32, 64])
            rot = rng.choice([0, 2, dim // 2, dim])
            layers.append(_parallel((kv * rng.choice([1, 2, 4]), kv, dim, rng.choice([4, 20, 32, 64]), rng.choice([1, 2, 3, 4]), round(rng.uniform(0.05, 0.5), 3),
                                     rot - rot % 2, rng.choice([100.0, 10000.0, 300000.0])),
                                    (rng.choice([1, 2, 4]), rng.choice([6, 16, 40]), rng.choice([7, 16, 64]), rng.choice([3.0, 15.0])),
                                    (round(rng.uniform(0.4, 1.5), 2), round(rng.uniform(0.4, 1.5), 2)), mlp()))
    return {"architecture": "Pekarax", "vocab": rng.choice([53, 128, 301]), "width": width, "norm": {"eps": rng.choice([1e-5, 1e-6, 1e-3])},
            "postln_alpha": rng.choice([1.0, 2.0, 3.5]), "layers": layers}


@pytest.mark.parametrize("seed", list(range(12)))
def test_drawn_configurations(tmp_path_factory, seed):
    from infinicore_infer_amd.engine import Engine
    cfg = _drawn_config(seed)
    folder = os.path.join(str(tmp_path_factory.getbasetemp()), "pekarax_drawn_%d" % seed)
    W = _write_model(folder, cfg, seed)
    rng = random.Random(seed + 100)
    requests = {"r%d" % i: H.random_tokens(cfg["vocab"], n, seed * 10 + i)
                for i, n in enumerate([rng.choice([1, 2, 5, 40, 66, 129, 150]) for _ in range(5)])}
    ref = {rid: P.forward(cfg, W, toks, torch.float64) for rid, toks in requests.items()}
    rounded = {rid: P.forward(cfg, W, toks, torch.float64, rnd=lambda x: x.to(torch.bfloat16).to(torch.float64)) for rid, toks in requests.items()}
    steps, max_tokens = H.trace_mixed(requests, seed=seed)
    for dname, dtype, tol in DTYPES:
        engine = Engine.from_dir(folder, dtype=dtype, max_tokens=max_tokens, page_size=16, max_requests=4)
        _compare(H.run_trace(engine, steps), ref, dtype, tol if dtype == torch.float32 else 0.3, "drawn %d %s" % (seed, dname), steps, rounded)
        engine.cache.check_invariants()
        assert not engine.cache.requests
