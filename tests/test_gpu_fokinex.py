"""The Fokinex decoder in the engine against the plain implementation of its equations (plain_fokinex.py): each mechanism's
kernel alone, then whole models in the four replay modes and both dtypes, with sizes, counts, constants and layer orders that
differ from model to model, and greedy generation through the entry point."""
import json
import math
import os
import random

import pytest
import torch

import helpers as H
import plain_fokinex as P

pytestmark = pytest.mark.gpu

DTYPES = [("float32", torch.float32, 1e-4), ("bfloat16", torch.bfloat16, 6e-2)]
NAN = float("nan")


def _i32(v):
    return torch.tensor(list(v), dtype=torch.int32, device="cuda")


def _latent(heads, dim, rot_dim, vdim, q_rank, kv_rank, scale, window, rot, kv_from=None, ff=None):
    """rot: (base, None or (factor, original, fast, slow))."""
    r = {"base": rot[0], "dims": rot_dim}
    if rot[1]:
        r["scaling"] = dict(zip(("factor", "original", "fast", "slow"), rot[1]))
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank, "scale": scale, "rot": r}
    if window:
        m["mask"] = {"size": window}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": m, "mlp": {"kind": "dense", "ff": ff} if ff else None}


def _parallel(left, right, scales, ff=None):
    """left: (heads, kv heads, dim, scale, softcap, window); right: (heads, kv heads, dim, vdim, conv)."""
    a = {"heads": left[0], "kv_heads": left[1], "dim": left[2], "vdim": left[2], "scale": left[3], "softcap": left[4]}
    if left[5]:
        a["mask"] = {"size": left[5]}
    b = dict(zip(("heads", "kv_heads", "dim", "vdim", "conv"), right))
    return {"type": "parallel", "mixer": {"left": a, "right": b, "left_scale": scales[0], "right_scale": scales[1]},
            "mlp": {"kind": "dense", "ff": ff} if ff else None}


# F1: a layer that reads another's rows over a LONGER window than that layer's own, and one that reads them with other heads and
# sizes over a shorter one; sizes of whole 16-byte pieces but no template's; stretched wavelengths with a ramp inside.
ROT1 = (10000.0, (4.0, 64, 8.0, 1.0))
F1 = {"architecture": "Fokinex", "vocab": 211, "width": 96, "norm": {"eps": 1e-5}, "embedding": {"scale": 7.0},
      "layers": [_latent(4, 24, 16, 40, 40, 64, 0.2, 37, ROT1, ff=112),
                 _parallel((4, 2, 40, 0.3, 3.0, 29), (4, 2, 24, 40, 4), (0.8, 1.3), ff=72),
                 _latent(3, 16, 16, 24, 24, 64, 0.25, 70, ROT1, kv_from=0, ff=56),
                 _latent(5, 24, 16, 32, 40, 64, 0.2, 18, ROT1, kv_from=0)]}
# F2: sizes that are no multiple of 4 or 8 (no tiled kernel takes them), no windows, no stretching, one tap, a single kv head and as
# many kv heads as heads, constants of one, a single-head latent layer, a reading layer right behind its source.
F2 = {"architecture": "Fokinex", "vocab": 97, "width": 70, "norm": {"eps": 1e-6}, "embedding": {"scale": 1.0},
      "layers": [_parallel((3, 3, 10, 0.4, 30.0, None), (3, 1, 6, 9, 1), (1.0, 1.0), ff=50),
                 _latent(1, 10, 6, 14, 18, 22, 0.3, None, (77.0, None), ff=33),
                 _latent(3, 5, 6, 7, 9, 22, 1.0, None, (77.0, None), kv_from=1),
                 _parallel((2, 1, 14, 1.0, 5.0, 3), (2, 2, 5, 3, 2), (1.0, -0.5))]}
# F3: the tiled kernels' sizes, windows that are multiples of a page, large head sizes in the recurrence, five taps, a source
# that keeps everything because one of its readers does.
ROT3 = (300000.0, (16.0, 32, 4.0, 0.5))
F3 = {"architecture": "Fokinex", "vocab": 300, "width": 128, "norm": {"eps": 1e-5}, "embedding": {"scale": 0.5},
      "layers": [_latent(4, 64, 32, 64, 64, 128, 0.1, 64, ROT3, ff=192),
                 _latent(6, 32, 32, 128, 48, 128, 0.15, None, ROT3, kv_from=0, ff=128),
                 _parallel((6, 2, 128, 0.09, 50.0, 48), (4, 1, 128, 64, 5), (1.1, 0.9), ff=64),
                 _parallel((5, 5, 64, 0.125, 8.0, 130), (2, 2, 64, 136, 3), (0.5, 1.5))]}
CONFIGS = {"F1": F1, "F2": F2, "F3": F3}
LENGTHS = {"F1": [1, 2, 130, 61, 210, 37], "F2": [3, 75, 1, 140, 18, 66], "F3": [2, 90, 17, 1, 300, 64]}


def _write_model(folder, cfg, seed):
    from safetensors.torch import save_file
    os.makedirs(folder, exist_ok=True)
    W = P.random_weights(cfg, seed)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file({k: v.to(torch.bfloat16).contiguous() for k, v in W.items()}, os.path.join(folder, "model.safetensors"))
    return W


_models, _engines, _plain = {}, {}, {}


def _model(tmp_path_factory, name):
    if name not in _models:
        folder = os.path.join(str(tmp_path_factory.getbasetemp()), "fokinex_" + name)
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


_rounding = {}


def _bf16_tolerance(cfg, W, requests, ref, least=6e-2):
    """What a bfloat16 run may differ by: three times what rounding the sublayers' inputs and results to 16 bits moves the plain
    implementation's logits by where that is most (values that nearly cancel before a norm magnify rounding)."""
    most = 0.0
    for rid, toks in requests.items():
        rounded = P.forward(cfg, W, toks, torch.float64, rnd=lambda x: x.to(torch.bfloat16).to(torch.float64))
        most = max(most, float((rounded - ref[rid]).abs().max()) / float(ref[rid].abs().max()))
    return max(least, 3 * most)


def _tolerance(tmp_path_factory, name, requests, dtype, tol):
    if dtype == torch.float32:
        return tol
    key = (name, tuple(requests))
    if key not in _rounding:
        _rounding[key] = _bf16_tolerance(CONFIGS[name], _model(tmp_path_factory, name)[1], requests, _reference(tmp_path_factory, name, requests))
    return _rounding[key]


MODES = {
    "whole": H.trace_whole,
    "tail": lambda r: H.trace_last_one_by_one(r, tail=100),     # long decoding: states move on token by token, windows pass
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
    tol = _tolerance(tmp_path_factory, name, requests, dtype, tol)
    got = H.run_trace(engine, steps)
    assert len(got) == sum(len(t) for t in requests.values())
    worst = H.compare(got, ref, tol, "%s %s %s" % (name, dname, mode), steps)
    print("worst error %.3g at %s (allowed %.3g)" % (worst[0], worst[1], tol))
    engine.cache.check_invariants()
    assert not engine.cache.requests
    for g in range(len(engine.groups)):
        assert engine.cache.free_pages(g) == engine.num_pages


def test_a_portion_does_not_depend_on_how_its_keys_are_made(tmp_path_factory, monkeypatch):
    """bfloat16 portions of latent attention over keys and values made per head, and (no memory for them) as matrix products over
    the latent rows: the same logits within rounding, also for portions that begin in the middle of a page."""
    from infinicore_infer_amd.parts import latent_attention
    requests = {"a": H.random_tokens(300, 300, 1), "b": H.random_tokens(300, 120, 2)}
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": requests["a"][:75], "want": list(range(75))}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": requests["a"][75:250], "want": list(range(175))},
                                     {"id": "b", "tokens": requests["b"], "want": list(range(120))}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": requests["a"][250:], "want": list(range(50))}], "end": ["a", "b"]}]
    ref = _reference(tmp_path_factory, "F3", requests)
    calls, real = [], latent_attention.LatentAttention._portion_by_products
    monkeypatch.setattr(latent_attention.LatentAttention, "_portion_by_products", lambda self, *a: (calls.append(1), real(self, *a))[1])
    for limit in (latent_attention.MADE_KEYS_BYTES, 0):
        monkeypatch.setattr(latent_attention, "MADE_KEYS_BYTES", limit)
        H.compare(H.run_trace(_engine(tmp_path_factory, "F3", torch.bfloat16, 1024), steps), ref, 6e-2, "limit %d" % limit, steps)
        assert len(calls) == (0 if limit else 8)


# ---- the comparison is sharp enough -------------------------------------------------------------------------------------
SHARP = json.loads(json.dumps(F1))
SHARP["norm"]["eps"] = 1e-2                      # so that the size of what a norm gets counts


def _with_weights(monkeypatch, change):
    """The plain implementation on changed weights: ``change(name, tensor)``."""
    real = P.forward
    monkeypatch.setattr(P, "forward", lambda cfg, W, tokens, dtype=torch.float64, **kw: real(
        cfg, {k: change(k, v) for k, v in W.items()}, tokens, dtype, **kw))


def _with_config(monkeypatch, change):
    real = P.forward

    def changed(cfg, W, tokens, dtype=torch.float64, **kw):
        cfg = json.loads(json.dumps(cfg))
        change(cfg)
        return real(cfg, W, tokens, dtype, **kw)
    monkeypatch.setattr(P, "forward", changed)


def _without_norm(monkeypatch, name, which=None):
    """One function with its unit_rms calls (or the ``which``-th) left out."""
    real, unit = getattr(P, name), P.unit_rms

    def bare(*a):
        calls = [0]

        def maybe(x, eps):
            calls[0] += 1
            return x if which is None or calls[0] == which + 1 else unit(x, eps)
        monkeypatch.setattr(P, "unit_rms", maybe)
        try:
            return real(*a)
        finally:
            monkeypatch.setattr(P, "unit_rms", unit)
    monkeypatch.setattr(P, name, bare)


def _tied(values="projected", bias="behind the cap", slope=lambda h, H_: 2.0 ** (-8.0 * (h + 1) / H_), gate=True, norm="row"):
    def attention(h, W, p, m, eps):
        T, H_, dim, G = h.shape[0], m["heads"], m["dim"], m["kv_heads"]
        raw = h @ W[p + "k"].T
        if norm == "row":
            q, k = P.unit_rms(h @ W[p + "q"].T, eps) * W[p + "q.norm"], P.unit_rms(raw, eps) * W[p + "k.norm"]
        else:
            q = P.unit_rms((h @ W[p + "q"].T).reshape(T, H_, dim), eps).reshape(T, -1) * W[p + "q.norm"]
            k = P.unit_rms(raw.reshape(T, G, dim), eps).reshape(T, -1) * W[p + "k.norm"]
        q, k = q.reshape(T, H_, dim), k.reshape(T, G, dim)
        v = k if values == "normed" else raw.reshape(T, G, dim)
        seen = P.seen_keys(T, m["mask"]["size"])
        back = (torch.arange(T)[:, None] - torch.arange(T)[None, :]).to(h.dtype)
        out = []
        for hd in range(H_):
            g = hd // (H_ // G)
            s, b, c = (q[:, hd] @ k[:, g].T) * m["scale"], slope(hd, H_) * back, m["softcap"]
            s = c * torch.tanh((s - b) / c) if bias == "before the cap" else c * torch.tanh(s / c) - b
            out.append(torch.softmax(s.masked_fill(~seen, -math.inf), -1) @ v[:, g])
        o = torch.cat(out, -1)
        return ((o * torch.sigmoid(h @ W[p + "g"].T)) if gate else o) @ W[p + "o"].T
    return attention


def _delta_memory(order):
    def memory(q, k, v, decay, beta):
        T, heads, dim = q.shape
        S = torch.zeros(heads, dim, v.shape[2], dtype=q.dtype)
        out = torch.zeros(T, heads, v.shape[2], dtype=q.dtype)
        read = lambda S, x: (S * x[:, :, None]).sum(1)
        for t in range(T):
            g, b = decay[t][:, None, None], beta[t][:, None]
            if order == "read first":
                S = g * S
                out[t] = read(S, q[t])
                S = S + k[t][:, :, None] * (b * (v[t] - read(S, k[t])))[:, None, :]
                continue
            if order == "error before the decay":
                u = b * (v[t] - read(S, k[t]))
                S = g * S + k[t][:, :, None] * u[:, None, :]
            elif order == "decay last":
                S = g * (S + k[t][:, :, None] * (b * (v[t] - read(S, k[t])))[:, None, :])
            elif order == "no delta rule":
                S = g * S + k[t][:, :, None] * (b * v[t])[:, None, :]
            else:                                           # no step size
                S = g * S
                S = S + k[t][:, :, None] * (v[t] - read(S, k[t]))[:, None, :]
            out[t] = read(S, q[t])
        return out
    return memory


def _serial(cfg, W, tokens, dtype=torch.float64, **kw):
    """The feed-forward reads the stream behind the mixer."""
    W, eps = {k: v.to(dtype) for k, v in W.items()}, cfg["norm"]["eps"]
    x, kept = W["embed"][torch.as_tensor(list(tokens))] * cfg["embedding"]["scale"], {}
    for i, l in enumerate(cfg["layers"]):
        p, m = "l%d." % i, l["mixer"]
        h = P.unit_rms(x, eps) * W[p + "norm1"]
        if l["type"] == "latent_attention":
            if m.get("kv_from") is None:
                kept[i] = P.latent_rows(h, W, p + "mix.", m, eps)
            x = x + P.latent_attention(h, W, p + "mix.", m, eps, kept[m.get("kv_from", i)])
        else:
            x = x + P.parallel_mixer(h, W, p + "mix.", m, eps)
        if l.get("mlp"):
            x = x + P.gated_unit(P.unit_rms(x, eps) * W[p + "norm1"], W, p + "mlp.")
    return (P.unit_rms(x, eps) * W["final.norm"]) @ W["head"].T


def _misread(monkeypatch, what):
    """One plausible misreading put into the plain implementation."""
    put = lambda name, f: monkeypatch.setattr(P, name, f)
    latents = lambda c: [l["mixer"] for l in c["layers"] if l["type"] == "latent_attention"]
    left = lambda c: c["layers"][1]["mixer"]["left"]
    freq, conv, rows = P.stretched_frequencies, P.short_conv, P.latent_rows
    if what == "the feed-forward behind the mixer":
        put("forward", _serial)
    elif what == "no embedding scale":
        _with_config(monkeypatch, lambda c: c["embedding"].update(scale=1.0))
    elif what == "norm weights around one":
        _with_weights(monkeypatch, lambda k, v: 1.0 + v if k.endswith("norm1") else v)
    elif what == "the query latent not normed":
        _without_norm(monkeypatch, "latent_attention", 0)
    elif what == "the key latent not normed":
        _without_norm(monkeypatch, "latent_rows", 0)
    elif what == "the rotated part normed":
        put("latent_rows", lambda h, W, p, m, eps: (rows(h, W, p, m, eps)[0], P.unit_rms(rows(h, W, p, m, eps)[1], eps)))
    elif what == "another layer's part before its rotation":
        real = P.latent_attention
        put("latent_attention", lambda h, W, p, m, eps, r: real(h, W, p, m, eps, r if m.get("kv_from") is None else (
            r[0], P.rotate_pairs(r[1], range(h.shape[0]), m["rot"]))))
    elif what == "halves rotated":
        def halves(x, positions, rot):
            d = rot["dims"]
            y = torch.cat([x[..., i::d // 2] for i in range(d // 2)], -1)                 # pairs (i, i + d/2) side by side
            z = real(y, positions, rot)
            out = x.clone()
            for i in range(d // 2):
                out[..., i], out[..., i + d // 2] = z[..., 2 * i], z[..., 2 * i + 1]
            return out
        real = P.rotate_pairs
        put("rotate_pairs", halves)
    elif what == "wavelengths not stretched":
        put("stretched_frequencies", lambda d, b, s=None: (freq(d, b)[0], freq(d, b, s)[1]))
    elif what == "all wavelengths stretched":
        put("stretched_frequencies", lambda d, b, s=None: ([f / s["factor"] for f in freq(d, b)[0]], freq(d, b, s)[1]))
    elif what == "no factor on cos and sin":
        put("stretched_frequencies", lambda d, b, s=None: (freq(d, b, s)[0], 1.0))
    elif what == "the factor on the whole score":
        real = P.latent_attention
        mult = freq(16, *[F1["layers"][0]["mixer"]["rot"][k] for k in ("base", "scaling")])[1]
        put("stretched_frequencies", lambda d, b, s=None: (freq(d, b, s)[0], 1.0))
        put("latent_attention", lambda h, W, p, m, eps, r: real(h, W, p, dict(m, scale=m["scale"] * mult * mult), eps, r))
    elif what == "fast and slow swapped":
        put("stretched_frequencies", lambda d, b, s=None: freq(d, b, dict(s, fast=s["slow"], slow=s["fast"])))
    elif what == "the ramp ends are not rounded":
        def exact(d, b, s=None):
            index = lambda t: d * math.log(s["original"] / (2 * math.pi * t)) / (2 * math.log(b))
            lo, hi = index(s["fast"]), index(s["slow"])
            ramp = [min(max((i - lo) / (hi - lo), 0.0), 1.0) for i in range(d // 2)]
            return [f / s["factor"] * r + f * (1 - r) for f, r in zip(freq(d, b)[0], ramp)], freq(d, b, s)[1]
        put("stretched_frequencies", exact)
    elif what == "scores over the root of the size":
        _with_config(monkeypatch, lambda c: [m.update(scale=(m["dim"] + m["rot_dim"]) ** -0.5) for m in latents(c)])
    elif what in ("a window one longer", "a window one shorter"):
        d = 1 if "longer" in what else -1
        _with_config(monkeypatch, lambda c: [m["mask"].update(size=m["mask"]["size"] + d) for m in latents(c)])
    elif what in ("the left window one longer", "the left window one shorter"):
        d = 1 if "longer" in what else -1
        _with_config(monkeypatch, lambda c: left(c)["mask"].update(size=left(c)["mask"]["size"] + d))
    elif what == "a reading layer with its source's window":
        _with_config(monkeypatch, lambda c: c["layers"][2]["mixer"]["mask"].update(size=37))
    elif what == "a source with its reader's window":
        _with_config(monkeypatch, lambda c: c["layers"][0]["mixer"]["mask"].update(size=70))
    elif what == "no sink":
        _with_weights(monkeypatch, lambda k, v: torch.full_like(v, -1e9) if k.endswith(".sink") else v)
    elif what == "a sink of zero":
        _with_weights(monkeypatch, lambda k, v: torch.zeros_like(v) if k.endswith(".sink") else v)
    elif what == "a scaled sink":
        real = P.softmax_with_sink
        put("softmax_with_sink", lambda s, sink=None: real(s, None if sink is None else sink * 0.2))
    elif what == "a sink on the left":
        real = P.softmax_with_sink
        put("softmax_with_sink", lambda s, sink=None: real(s, torch.zeros((), dtype=s.dtype) if sink is None else sink))
    elif what == "values normed like the keys":
        put("tied_attention", _tied(values="normed"))
    elif what == "norms per head":
        put("tied_attention", _tied(norm="head"))
    elif what == "no cap":
        _with_config(monkeypatch, lambda c: left(c).update(softcap=1e9))
    elif what == "the distance bias before the cap":
        put("tied_attention", _tied(bias="before the cap"))
    elif what == "no distance bias":
        put("tied_attention", _tied(slope=lambda h, H_: 0.0))
    elif what == "slopes from zero":
        put("tied_attention", _tied(slope=lambda h, H_: 2.0 ** (-8.0 * h / H_)))
    elif what == "no gate on the left":
        put("tied_attention", _tied(gate=False))
    elif what in ("read first", "error before the decay", "decay last", "no delta rule", "no step size"):
        put("delta_memory", _delta_memory(what))
    elif what == "queries and keys not of unit length":
        put("unit_length", lambda x: x)
    elif what == "unit root mean square instead of unit length":
        put("unit_length", lambda x: P.unit_rms(x, 1e-6))
    elif what == "taps in reverse":
        put("short_conv", lambda x, w: conv(x, w.flip(1)))
    elif what == "the convolution sees one token less":
        put("short_conv", lambda x, w: conv(x, torch.cat([torch.zeros_like(w[:, :1]), w[:, 1:]], 1)))
    elif what == "heads share query/key heads in turn":
        real = torch.Tensor.repeat_interleave
        monkeypatch.setattr(torch.Tensor, "repeat_interleave", lambda x, n, d: x.repeat(1, n, 1) if d == 1 else real(x, n, d))
    elif what == "decay rate not exponentiated":
        _with_weights(monkeypatch, lambda k, v: torch.log(v.abs() + 1e-9) if k.endswith(".A_log") else v)
    elif what == "no bias on the decay":
        _with_weights(monkeypatch, lambda k, v: torch.zeros_like(v) if k.endswith(".dt_bias") else v)
    elif what == "no norm on the recurrence's result":
        _without_norm(monkeypatch, "delta_mixer", 0)
    elif what == "a sigmoid gate on the right":
        real_silu, real = P.silu, P.delta_mixer

        def gated(h, W, p, m, eps):
            calls = [0]

            def silu(z):
                calls[0] += 1
                return torch.sigmoid(z) if calls[0] == 4 else real_silu(z)
            monkeypatch.setattr(P, "silu", silu)
            try:
                return real(h, W, p, m, eps)
            finally:
                monkeypatch.setattr(P, "silu", real_silu)
        put("delta_mixer", gated)
    elif what == "no scale on the left":
        _with_config(monkeypatch, lambda c: c["layers"][1]["mixer"].update(left_scale=1.0))
    elif what == "no scale on the right":
        _with_config(monkeypatch, lambda c: c["layers"][1]["mixer"].update(right_scale=1.0))
    else:
        raise ValueError(what)


MISREADINGS = [
    "the feed-forward behind the mixer", "no embedding scale", "norm weights around one", "the query latent not normed",
    "the key latent not normed", "the rotated part normed", "another layer's part before its rotation", "halves rotated",
    "wavelengths not stretched", "all wavelengths stretched", "no factor on cos and sin", "the factor on the whole score",
    "fast and slow swapped", "the ramp ends are not rounded", "scores over the root of the size", "a window one longer",
    "a window one shorter", "the left window one longer", "the left window one shorter", "a reading layer with its source's window",
    "a source with its reader's window", "no sink", "a sink of zero", "a scaled sink", "a sink on the left",
    "values normed like the keys", "norms per head", "no cap", "the distance bias before the cap", "no distance bias",
    "slopes from zero", "no gate on the left", "read first", "error before the decay", "decay last", "no delta rule", "no step size",
    "queries and keys not of unit length", "unit root mean square instead of unit length", "taps in reverse",
    "the convolution sees one token less", "heads share query/key heads in turn", "decay rate not exponentiated",
    "no bias on the decay", "no norm on the recurrence's result", "a sigmoid gate on the right", "no scale on the left",
    "no scale on the right"]


@pytest.fixture(scope="module")
def sharp_run(tmp_path_factory):
    """One request through the float32 engine: the misreadings are held against its logits."""
    from infinicore_infer_amd.engine import Engine
    folder = os.path.join(str(tmp_path_factory.getbasetemp()), "fokinex_sharp")
    W = _write_model(folder, SHARP, 33)
    toks = H.random_tokens(F1["vocab"], 120, 21)
    engine = Engine.from_dir(folder, dtype=torch.float32, max_tokens=128, page_size=16, max_requests=1)
    steps, _ = H.trace_whole({"a": toks})
    got = H.run_trace(engine, steps)
    H.compare(got, {"a": P.forward(SHARP, W, toks, torch.float64)}, 1e-4, "as designed")
    return W, toks, got


@pytest.mark.parametrize("what", MISREADINGS)
def test_a_misreading_of_the_design_shows(sharp_run, monkeypatch, what):
    """The comparison the other tests rest on is sharp enough: with one misreading in the plain implementation the float32
    engine no longer agrees with it (the same request agrees without)."""
    W, toks, got = sharp_run
    _misread(monkeypatch, what)
    with pytest.raises(AssertionError):
        H.compare(got, {"a": P.forward(SHARP, W, toks, torch.float64)}, 1e-4, what)


def test_the_residual_stream_after_every_layer(tmp_path_factory):
    """Layer by layer in float32: the stream after every layer, with what the layer still owes it."""
    from infinicore_infer_amd.engine import Engine, StepEntry
    folder, W = _model(tmp_path_factory, "F3")
    toks = H.random_tokens(F3["vocab"], 75, 3)
    want = []
    P.forward(F3, W, toks, torch.float64, layers_out=want)
    eng = Engine.from_dir(folder, dtype=torch.float32, max_tokens=128, max_requests=1)
    got, build = [], eng._build_context

    def probe(i, x, pending):
        x = x.clone()
        for y, f in getattr(pending, "parts", ()):
            x += f * y
        got.append(x)

    def probed(entries, starts):
        ctx = build(entries, starts)
        ctx.layer_probe = probe
        return ctx
    eng._build_context = probed
    eng.step([StepEntry("a", toks, [])])
    assert len(want) == 4 and len(got) >= 4
    for i, w in enumerate(want):
        assert torch.allclose(got[i].cpu().double(), w, atol=2e-5 * float(w.abs().max())), "after layer %d" % i


@pytest.mark.parametrize("name,page_size", [("F1", 64), ("F3", 32)])
def test_other_page_sizes(tmp_path_factory, name, page_size):
    requests = _requests(name, seed=2)
    steps, max_tokens = H.trace_mixed(requests, seed=5)
    ref = _reference(tmp_path_factory, name, requests)
    for dtype, tol in ((torch.float32, 1e-4), (torch.bfloat16, 6e-2)):
        engine = _engine(tmp_path_factory, name, dtype, max_tokens + 4 * page_size, page_size=page_size)
        H.compare(H.run_trace(engine, steps), ref, tol, "%s page %d" % (name, page_size))
        engine.cache.check_invariants()


@pytest.mark.parametrize("dtype,tol", [(torch.float32, 1e-4), (torch.bfloat16, 6e-2)])
@pytest.mark.parametrize("name", ["F1", "F3"])
def test_recorded_decode_steps_equal_eager_ones(tmp_path_factory, name, dtype, tol):
    """Long decoding: the same request decoded through recorded steps and eagerly gives the same logits; states and convolution
    inputs move on exactly once per step, also in the step that is recorded, and windows give their pages back meanwhile."""
    from infinicore_infer_amd.engine import Engine, StepEntry
    folder, W = _model(tmp_path_factory, name)
    cfg = CONFIGS[name]
    toks = H.random_tokens(cfg["vocab"], 330, 9)
    rows = {}
    for graphs in (True, False):
        eng = Engine.from_dir(folder, dtype=dtype, max_tokens=512, page_size=16, max_requests=2, use_graphs=graphs)
        eng.step([StepEntry("a", toks[:30], [])])
        out = []
        for t in toks[30:]:
            out.append(eng.step([StepEntry("a", [t], [0])]).float().cpu().clone())
        rows[graphs] = torch.cat(out)
        if graphs:
            assert eng.graph_replays > 200
        # a window group holds no more pages than its window spans
        for g, spec in enumerate(eng.groups):
            held = sum(p >= 0 for p in eng.cache.block_table("a", g))
            assert held <= (spec.window + 15) // 16 + 1 if spec.kind == "window" else held == 21
    assert torch.equal(rows[True], rows[False])
    ref = P.forward(cfg, W, toks, torch.float64)[30:]
    assert float((rows[True].double() - ref).abs().max()) <= tol * float(ref.abs().max())


def test_a_forked_request_goes_on_apart(tmp_path_factory):
    """A copy of a request (its pages and its states) and the original continue with different tokens."""
    from infinicore_infer_amd.engine import Engine, StepEntry
    folder, W = _model(tmp_path_factory, "F1")
    toks = H.random_tokens(F1["vocab"], 90, 11)
    a_tail, b_tail = H.random_tokens(F1["vocab"], 30, 12), H.random_tokens(F1["vocab"], 30, 13)
    eng = Engine.from_dir(folder, dtype=torch.float32, max_tokens=512, page_size=16, max_requests=3, use_graphs=False)
    eng.step([StepEntry("a", toks, [])])
    eng.fork("a", "b")
    la = eng.step([StepEntry("a", a_tail, list(range(30)))]).float().cpu().clone()
    lb = eng.step([StepEntry("b", b_tail, list(range(30)))]).float().cpu().clone()
    for got, tail in ((la, a_tail), (lb, b_tail)):
        ref = P.forward(F1, W, toks + tail, torch.float64)[90:]
        assert float((got.double() - ref).abs().max()) <= 1e-4 * float(ref.abs().max())
    eng.free("a")
    eng.free("b")
    eng.cache.check_invariants()


@pytest.mark.parametrize("rows", [1, 3, 16, 17, 40, 64])
def test_few_rows_take_fused_products_and_give_the_same_logits(tmp_path_factory, rows):
    """A decode step of 1..64 requests at sizes where the last projections add to the stream in their epilogues (up to 16
    rows) or run in slices that take the mixers' results along (17..64), against library products and a row kernel."""
    from infinicore_infer_amd.engine import Engine, StepEntry
    from infinicore_infer_amd.kernels import ops
    name = "wide"
    if name not in CONFIGS:
        CONFIGS[name] = {"architecture": "Fokinex", "vocab": 160, "width": 1024, "norm": {"eps": 1e-5}, "embedding": {"scale": 2.0},
                         "layers": [_latent(8, 64, 32, 64, 256, 256, 0.1, 40, ROT3, ff=4096),
                                    _parallel((16, 4, 64, 0.125, 30.0, 24), (16, 4, 64, 64, 4), (0.7, 1.2), ff=4096),
                                    _latent(8, 64, 32, 64, 256, 256, 0.1, 90, ROT3, kv_from=0)]}
    folder, W = _model(tmp_path_factory, name)
    prompts = [H.random_tokens(160, 5 + 3 * (i % 9), 60 + i) for i in range(rows)]
    tails = [H.random_tokens(160, 3, 160 + i) for i in range(rows)]
    out = {}
    for impl in ("auto", "library"):
        key = ("wide", impl)
        if key not in _engines:
            _engines[key] = Engine.from_dir(folder, dtype=torch.bfloat16, max_tokens=64 * 64, page_size=16, max_requests=64, gemm_impl=impl)
        eng = _engines[key]
        assert ops.rule_tail(torch.bfloat16, *(torch.empty(n, 4096, dtype=torch.bfloat16) for n in (rows, 1024))) == (
            ops.TAIL_SPLIT_NORM if rows <= 16 else ops.TAIL_SLICES)
        for i, p in enumerate(prompts):
            eng.step([StepEntry(i, p, [])])
        got = [eng.step([StepEntry(i, [t[j]], [0]) for i, t in enumerate(tails)]).float().cpu().clone() for j in range(3)]
        for i in range(rows):
            eng.free(i)
        out[impl] = torch.stack(got)
    scale = float(out["library"].abs().max())
    assert float((out["auto"] - out["library"]).abs().max()) <= 3e-2 * scale
    for i in sorted({0, rows - 1}):
        ref = P.forward(CONFIGS[name], W, prompts[i] + tails[i], torch.float64)[-3:]
        assert float((out["auto"][:, i].double() - ref).abs().max()) <= 6e-2 * float(ref.abs().max())


# ---- each mechanism's kernel alone ----------------------------------------------------------------------------------------
def _close(got, want, tol, what):
    err = float((got.float().cpu().double() - want).abs().max()) / max(1e-6, float(want.abs().max()))
    assert math.isfinite(err) and err <= tol, "%s: error %.3g (allowed %.3g)" % (what, err, tol)


@pytest.mark.parametrize("dims,base,scaling", [(16, 10000.0, (4.0, 64, 8.0, 1.0)), (64, 1e6, (32.0, 4096, 32.0, 1.0)), (6, 77.0, None),
                                               (24, 3e5, (6.0, 100, 2.0, 2.0)), (8, 100.0, (2.0, 3, 50.0, 0.01)), (2, 10.0, (3.0, 512, 32.0, 1.0))])
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_rotation_with_stretched_wavelengths(dtype, dims, base, scaling):
    """The cached row (normed latent, rotated part) and the queries' rotated parts, into another tensor and in place, at
    positions up to 60,000: angles as exact there as at the start, the factor on cos and sin, the rest passing unchanged."""
    from infinicore_infer_amd.kernels import ops
    from infinicore_infer_amd.parts.rotary import pair_frequencies, stretched_magnitude
    s = dict(zip(("factor", "original", "fast", "slow"), scaling)) if scaling else None
    rot = {"base": base, "dims": dims, "scaling": s}
    freq = pair_frequencies(dims, base, s)
    want_f, mult = P.stretched_frequencies(dims, base, s)
    assert torch.allclose(freq.double().sum(0), torch.tensor(want_f, dtype=torch.float64), rtol=1e-12) and stretched_magnitude(s) == mult
    E, R, Rq, dim, Hn, eps, page = dims + 4, 24, 20, 10, 3, 1e-5, 16
    pos = [0, 1, 2, 17, 100, 1023, 4097, 33333, 60000]
    T = len(pos)
    g = torch.Generator().manual_seed(dims)
    rows = torch.randn(T, Rq + R + E, generator=g).to(dtype)
    qn, kn = 1 + 0.2 * torch.randn(Rq, generator=g), 1 + 0.2 * torch.randn(R, generator=g)
    slots = _i32([5, 40, 3, 17, 16, 31, 0, 63, 22])
    cache = torch.zeros(4, 1, page, R + E, dtype=dtype, device="cuda")
    cq = torch.empty(T, Rq, dtype=dtype, device="cuda")
    ops.latent_prep(rows.cuda(), Rq, R, E, qn.cuda(), kn.cuda(), eps, freq.cuda(), dims, _i32(pos), cq, cache, slots, mult)
    r64, tol = rows.double(), 1e-5 if dtype == torch.float32 else 2e-2
    assert torch.allclose(cq.cpu().double(), P.unit_rms(r64[:, :Rq], eps) * qn.double(), atol=tol)
    flat = cache.view(-1, R + E).cpu().double()[slots.long().cpu()]
    assert torch.allclose(flat[:, :R], P.unit_rms(r64[:, Rq:Rq + R], eps) * kn.double(), atol=tol)
    assert torch.allclose(flat[:, R:], P.rotate_pairs(r64[:, Rq + R:], pos, rot), atol=tol)
    # a layer that caches nothing: only the query latent
    cq2 = torch.full_like(cq, NAN)
    ops.latent_prep(rows[:, :Rq].contiguous().cuda(), Rq, R, E, qn.cuda(), None, eps, freq.cuda(), dims, _i32(pos), cq2, None, None, mult)
    assert torch.equal(cq, cq2)
    q = torch.randn(T, Hn * (dim + E), generator=g).to(dtype)
    want = P.rotate_pairs(q.double().view(T, Hn, dim + E)[:, :, dim:], pos, rot)
    qa = torch.zeros(T, Hn * (R + E), dtype=dtype, device="cuda")
    ops.latent_q_rotate(q.cuda(), dim, E, R, Hn, freq.cuda(), dims, _i32(pos), qa, mult)
    got = qa.view(T, Hn, R + E).cpu().double()
    assert torch.allclose(got[:, :, R:], want, atol=4 * tol) and float(got[:, :, :R].abs().max()) == 0
    turned = q.cuda()
    ops.latent_q_rotate(turned, dim, E, dim, Hn, freq.cuda(), dims, _i32(pos), turned, mult)
    got = turned.view(T, Hn, dim + E).cpu()
    assert torch.equal(got[:, :, :dim], q.view(T, Hn, dim + E)[:, :, :dim]) and torch.allclose(got[:, :, dim:].double(), want, atol=4 * tol)


def _needle(q, row, score, scale):
    """``q`` replaced by a query whose score against ``row`` is ``score``."""
    return row * (score / scale / float(row.pow(2).sum()))


@pytest.mark.parametrize("R,E,Hn,page,window", [(64, 32, 6, 16, 40), (40, 8, 3, 16, 33), (22, 6, 2, 32, 1), (128, 64, 40, 64, 64),
                                                (512, 64, 4, 16, 100), (64, 16, 5, 16, 0)])
@pytest.mark.parametrize("dname,dtype,tol", DTYPES)
def test_walk_over_a_window_of_latent_rows_with_sinks(R, E, Hn, page, window, dname, dtype, tol):
    """Queries around page borders and key steps.  One head's query is aligned with the first key of its window, another's with the
    key just before it (which must count for nothing), a third's with its own key; every page that lies wholly outside the
    window, and every row beyond the position, holds NaN.  Keys split several ways, sinks that carry a good part of the weight."""
    from infinicore_infer_amd.kernels import ops
    D, scale = R + E, 0.5 / math.sqrt(R + E)
    g = torch.Generator().manual_seed(R + Hn)
    cases = [p for p in (0, 1, 15, 16, 31, 32, 33, 63, 64, 65, 100, 127, 128, 200, 299)]
    T, n_pages = len(cases), 300 // page + 1
    plane = torch.full((T * n_pages, 1, page, D), NAN)
    order = torch.randperm(T * n_pages, generator=g)
    bt = order.view(T, n_pages).to(torch.int32)
    sinks = torch.randn(Hn, generator=g) * 2 + 1
    q, want = torch.randn(T, Hn, D, generator=g), torch.zeros(T, Hn, R, dtype=torch.float64)
    for i, pos in enumerate(cases):
        lo = max(0, pos - window + 1) if window else 0
        rows = torch.randn(pos + 1, D, generator=g).to(dtype).float()
        q[i, 0] = _needle(q[i, 0], rows[lo], 6.0, scale)
        if lo > 0:
            q[i, 1] = _needle(q[i, 1], rows[lo - 1], 9.0, scale)
        q[i, Hn - 1] = _needle(q[i, Hn - 1], rows[pos], 6.0, scale)
        q[i] = q[i].to(dtype).float()
        for j in range(lo // page * page, pos + 1):                 # (rows of the window's first page that lie before it are real ones)
            plane[bt[i, j // page], 0, j % page] = rows[j]
        s = q[i].double() @ rows[lo:].double().T * scale
        p = P.softmax_with_sink(s, sinks.double()[:, None])
        want[i] = p @ rows[lo:, :R].double()
    qa = q.to(dtype).reshape(T, Hn * D).cuda()
    plane = plane.to(dtype).cuda()
    on_cores = ops.attention_latent_on_matrix_cores(dtype, R, E)
    for n_split, vector in [(1, False), (2, False), (7, False)] + ([(1, True), (3, True)] if on_cores else []):
        out = torch.full((T, Hn * R), NAN, dtype=dtype, device="cuda")
        acc = torch.empty(T * Hn * n_split * R, dtype=torch.float32, device="cuda")
        ml = torch.empty(T * Hn * n_split * 2, dtype=torch.float32, device="cuda")
        ops.attention_latent(qa, out, plane, bt.cuda(), _i32(range(T)), _i32(cases), Hn, R, E, page, scale, n_split, acc, ml,
                             vector_units=vector, window=window, sinks=sinks.cuda())
        err = (out.view(T, Hn, R).cpu().double() - want).abs().amax(dim=(1, 2)) / want.abs().max()
        assert float(err.max()) <= (2e-5 if dtype == torch.float32 else 2e-2), (n_split, vector, cases[int(err.argmax())], float(err.max()))


@pytest.mark.parametrize("dim,E,dv,R,Hn,window,with_gate", [(24, 16, 40, 64, 3, 37, False), (64, 32, 64, 256, 4, 0, True), (128, 64, 128, 512, 2, 129, False),
                                                            (40, 32, 72, 72, 5, 64, False), (56, 8, 96, 40, 2, 1, True), (80, 48, 128, 96, 2, 200, False),
                                                            (160, 32, 56, 64, 1, 63, False), (8, 8, 8, 8, 6, 5, False)])
@pytest.mark.parametrize("n,pos0", [(2, 0), (33, 0), (300, 0), (129, 171), (64, 64), (40, 299)])
def test_portions_over_keys_and_values_made_per_head(dim, E, dv, R, Hn, window, with_gate, n, pos0):
    """One request's portion on the matrix cores: queries whose score singles out the first key of their window or the key just
    before it, in tiles of 128 tokens, over steps of 64 keys, at positions that begin anywhere; NaN in all rows that
    nobody sees and in the token rows of other requests."""
    from infinicore_infer_amd.kernels import ops
    scale, g = 0.7 / math.sqrt(dim + E), torch.Generator().manual_seed(dim + n + pos0)
    L, first = pos0 + n, max(0, pos0 - window + 1) if window else 0
    key0, row0 = first // 16 * 16, 7
    keys = (L - key0 + 15) // 16 * 16
    bf = lambda *s: torch.randn(*s, generator=g).to(torch.bfloat16)
    k_plain, v, k_rot = bf(L, Hn, dim), bf(L, Hn, dv), bf(L, E)
    q = torch.randn(n, Hn, dim + E, generator=g)
    full = torch.cat([k_plain.float(), k_rot.float()[:, None].expand(L, Hn, E)], -1)
    for t in range(0, n, 5):
        lo = max(0, pos0 + t - window + 1) if window else 0
        q[t, 0] = _needle(q[t, 0], full[lo, 0], 7.0, scale)
        if lo > 0:
            q[t, Hn - 1] = _needle(q[t, Hn - 1], full[lo - 1, Hn - 1], 9.0, scale)
    q = q.to(torch.bfloat16)
    sinks = torch.randn(Hn, generator=g) * 2
    gate = bf(n, Hn * dv) if with_gate else None
    back = (pos0 + torch.arange(n))[:, None] - torch.arange(L)[None, :]
    seen = (back >= 0) & ((back < window) if window else True)
    want = torch.zeros(n, Hn, dv, dtype=torch.float64)
    for hd in range(Hn):
        s = (q[:, hd].double() @ full[:, hd].double().T) * scale
        want[:, hd] = P.softmax_with_sink(s.masked_fill(~seen, -math.inf), sinks.double()[hd]) @ v[:, hd].double()
    want = want.reshape(n, Hn * dv)
    if with_gate:
        want = want * torch.sigmoid(gate.double())
    kv = torch.full((keys, Hn * (dim + dv)), NAN, dtype=torch.bfloat16)
    rows = torch.full((keys, R + E), NAN, dtype=torch.bfloat16)
    a, b = first - key0, L - key0
    kv[a:b] = torch.cat([k_plain[first:].reshape(n + pos0 - first, -1), v[first:].reshape(n + pos0 - first, -1)], 1)
    rows[a:b, R:] = k_rot[first:]
    qs = torch.full((row0 + n + 3, Hn * (dim + E)), NAN, dtype=torch.bfloat16)
    qs[row0:row0 + n] = q.reshape(n, -1)
    out = torch.full((row0 + n + 3, Hn * dv), 5.0, dtype=torch.bfloat16, device="cuda")
    gs = None
    if with_gate:
        gs = torch.full((row0 + n + 3, Hn * dv + 8), NAN, dtype=torch.bfloat16)
        gs[row0:row0 + n, 8:] = gate
        gs = gs.cuda()[:, 8:]
    ops.attention_latent_prefill(qs.cuda(), out, gs, kv.cuda(), rows.cuda(), R, key0, row0, n, pos0, Hn, dim, E, dv, scale,
                                 window=window, sinks=sinks.cuda())
    got = out.cpu()
    assert bool((got[:row0] == 5.0).all()) and bool((got[row0 + n:] == 5.0).all())
    _close(got[row0:row0 + n], want, 1.5e-2, "portion of %d at %d" % (n, pos0))


@pytest.mark.parametrize("R,E,page,L,first", [(64, 32, 16, 150, 37), (40, 8, 32, 70, 33), (24, 6, 16, 47, 16), (128, 64, 64, 300, 0)])
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_gathered_rows_of_a_window_and_the_softmax_over_it(R, E, page, L, first, dtype):
    """A request's rows from a key on (zeros where they may have been given back), alone and with their transposed copy; the
    masked softmax of a portion whose columns begin at that key, with sinks."""
    from infinicore_infer_amd.kernels import ops
    D, Hn, key0 = R + E, 3, first // 16 * 16
    g = torch.Generator().manual_seed(L)
    n_pages = (L + page - 1) // page
    order = torch.randperm(n_pages + 2, generator=g)[:n_pages]
    rows = torch.randn(L, D, generator=g).to(dtype)
    plane = torch.full((n_pages + 2, 1, page, D), NAN, dtype=dtype)
    for j in range(first, L):
        plane[order[j // page], 0, j % page] = rows[j]
    bt = order.to(torch.int32).cuda()
    pad = (L - key0 + 15) // 16 * 16
    want = torch.zeros(pad, D, dtype=dtype)
    want[first - key0:L - key0] = rows[first:]
    for transposed in (True, False):
        got = torch.full((pad, D), NAN, dtype=dtype, device="cuda")
        got_t = torch.full((R, pad), NAN, dtype=dtype, device="cuda") if transposed else None
        ops.latent_gather(plane.cuda(), bt, L, pad, page, R, got, got_t, key0=key0, first=first)
        assert torch.equal(got.cpu(), want)
        assert not transposed or torch.equal(got_t.cpu(), want[:, :R].T)
    window = 21
    pos0 = first + window - 1                       # the portion's first token sees first .. pos0
    n = L - pos0
    if n <= 0:
        return
    sinks = torch.randn(Hn, generator=g)
    scores = torch.randn(n * Hn, pad, generator=g) * 3
    probs = torch.full((n * Hn, pad), NAN, dtype=dtype, device="cuda")
    ops.latent_softmax(scores.cuda(), probs, Hn, pos0, 0.37, window=window, sinks=sinks.cuda(), key0=key0)
    want = torch.zeros(n * Hn, pad, dtype=torch.float64)
    for m in range(n * Hn):
        pos = pos0 + m // Hn
        a, b = max(0, pos - window + 1) - key0, pos + 1 - key0
        want[m, a:b] = P.softmax_with_sink(scores[m, a:b].double() * 0.37, sinks.double()[m % Hn:m % Hn + 1])
    assert torch.allclose(probs.float().cpu().double(), want, atol=1e-6 if dtype == torch.float32 else 4e-3)


@pytest.mark.parametrize("Hq,G,d", [(4, 2, 40), (3, 3, 10), (6, 2, 128), (2, 1, 96), (5, 5, 64), (1, 1, 200)])
@pytest.mark.parametrize("mode", [0, 1, 2])
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_values_that_are_the_projected_keys(dtype, mode, Hq, G, d):
    """Rows [q | k | gate]: the cache's value plane holds the keys as projected (with their bias), its key plane the normed ones."""
    from infinicore_infer_amd.kernels import ops
    T, page, eps = 7, 16, 1e-5
    g = torch.Generator().manual_seed(d + mode)
    rows = torch.randn(T, (2 * Hq + G) * d, generator=g).to(dtype)
    bias = torch.randn((Hq + G) * d, generator=g) if d % 8 else None
    qw, kw = (None, None) if mode == 0 else (1 + 0.3 * torch.randn(n, generator=g) for n in ((d, d) if mode == 1 else (Hq * d, G * d)))
    kc, vc = (torch.zeros(3, G, page, d, dtype=dtype, device="cuda") for _ in range(2))
    q_out = torch.empty(T, Hq * d, dtype=dtype, device="cuda")
    slots = [0, 47, 17, 16, 15, 31, 32]
    dev = lambda t: None if t is None else t.cuda()
    ops.qk_norm_store(rows.cuda(), dev(bias), dev(qw), dev(kw), mode, eps, 0, None, None, q_out, kc, vc, _i32(slots), Hq, G, d, d, page,
                      values_from_keys=True)
    x = rows.double()[:, :(Hq + G) * d] + (bias.double() if bias is not None else 0.0)
    q, k = x[:, :Hq * d], x[:, Hq * d:]
    if mode == 1:
        unit = lambda z, n, w: (P.unit_rms(z.view(T, n, d), eps) * w.double()).reshape(T, -1)
        wq, wk = unit(q, Hq, qw), unit(k, G, kw)
    else:
        wq, wk = (q, k) if mode == 0 else (P.unit_rms(q, eps) * qw.double(), P.unit_rms(k, eps) * kw.double())
    tol = dict(atol=1e-5, rtol=1e-5) if dtype == torch.float32 else dict(atol=2e-2, rtol=1e-2)
    assert torch.allclose(q_out.cpu().double(), wq, **tol)
    for t, s in enumerate(slots):
        assert torch.allclose(kc[s // page, :, s % page].cpu().double(), wk[t].view(G, d), **tol)
        assert torch.allclose(vc[s // page, :, s % page].cpu().double(), k[t].view(G, d), **tol)
        assert bias is not None or torch.equal(vc[s // page, :, s % page].cpu(), rows[t, Hq * d:(Hq + G) * d].view(G, d))


@pytest.mark.parametrize("Hq,G,dk,dv,window,cap,page", [(6, 3, 96, 96, 33, 4.0, 16), (6, 2, 128, 128, 0, 50.0, 64), (3, 3, 40, 40, 17, 0.0, 16),
                                                        (8, 1, 64, 64, 64, 20.0, 16), (5, 5, 80, 48, 1, 3.0, 32), (2, 1, 24, 104, 100, 0.0, 16),
                                                        (2, 2, 10, 14, 20, 8.0, 16)])
@pytest.mark.parametrize("dname,dtype,tol", DTYPES)
def test_distance_bias_in_every_attention_kernel(dname, dtype, tol, Hq, G, dk, dv, window, cap, page):
    """slope_h (i - j) taken off the capped score, in the general kernel, the single tokens' (their keys split) and the prompt
    portions', for sizes with a kernel of their own and sizes between; queries aligned with the first key of their window and
    with the key just before it, NaN in every page that nobody sees; slopes from steep to none."""
    from infinicore_infer_amd.kernels import ops
    scale, lens = 0.8 / math.sqrt(dk), [300, 140, 7]
    g = torch.Generator().manual_seed(dk + window)
    slopes = torch.tensor([2.0 ** (-8.0 * (h + 1) / Hq) for h in range(Hq)])
    slopes[-1] = 0.0
    n_pages = [(n + page - 1) // page for n in lens]
    order = torch.randperm(sum(n_pages) + 3, generator=g).tolist()
    kc, vc = torch.full((len(order), G, page, dk), NAN), torch.full((len(order), G, page, dv), NAN)
    bt, K, V = torch.zeros(len(lens), max(n_pages), dtype=torch.int32), [], []
    for r, n in enumerate(lens):
        k, v = torch.randn(n, G, dk, generator=g).to(dtype), torch.randn(n, G, dv, generator=g).to(dtype)
        for j in range(n_pages[r]):
            bt[r, j] = order.pop()
        for j in range(n):
            kc[bt[r, j // page], :, j % page], vc[bt[r, j // page], :, j % page] = k[j].float(), v[j].float()
        K.append(k.float())
        V.append(v.double())
    kc, vc, bt = kc.to(dtype).cuda(), vc.to(dtype).cuda(), bt.cuda()

    def run(kernel, portions):
        qs, refs, req, pos, tiles, row = [], [], [], [], [], 0
        for r, p0, n in portions:
            q = torch.randn(n, Hq, dk, generator=g)
            lo = max(0, p0 + n - window) if window else 0
            q[n - 1, 0] = _needle(q[n - 1, 0], K[r][lo, 0], 7.0, scale)
            if lo > 0:
                q[n - 1, Hq - 1] = _needle(q[n - 1, Hq - 1], K[r][lo - 1, G - 1], 9.0, scale)
            q = q.to(dtype)
            back = ((p0 + torch.arange(n))[:, None] - torch.arange(lens[r])[None, :]).double()
            seen = (back >= 0) & ((back < window) if window else True)
            ref = torch.zeros(n, Hq, dv, dtype=torch.float64)
            for hd in range(Hq):
                kv = hd // (Hq // G)
                s = (q[:, hd].double() @ K[r][:, kv].double().T) * scale
                s = cap * torch.tanh(s / cap) if cap else s
                s = (s - float(slopes[hd]) * back).masked_fill(~seen, -math.inf)
                ref[:, hd] = torch.softmax(s, -1) @ V[r][:, kv]
            refs.append(ref.reshape(n, -1))
            qs.append(q.reshape(n, -1))
            req += [r] * n
            pos += range(p0, p0 + n)
            tiles += [(r, row + o, min(128, n - o), p0 + o) for o in range(0, n, 128)]
            row += n
        q = torch.cat(qs).cuda()
        out = torch.full((row, Hq * dv), NAN, dtype=dtype, device="cuda")
        args = (Hq, G, dk, dv, page, scale, window, 0, False, cap, slopes.cuda())
        if kernel == "general":
            ops.attention_span_generic(q, out, None, kc, vc, bt, _i32(req), _i32(pos), *args)
        elif kernel == "prefill":
            ops.attention_span_prefill(q, out, None, kc, vc, bt, torch.tensor(tiles, dtype=torch.int32).cuda(), len(tiles), *args)
        else:
            pa = torch.empty(row * Hq * kernel * dv, dtype=torch.float32, device="cuda")
            pm = torch.empty(row * Hq * kernel * 2, dtype=torch.float32, device="cuda")
            ops.attention_span_decode(q, out, None, kc, vc, bt, None, row, _i32(req), _i32(pos), pa, pm, *args, n_split=kernel)
        _close(out, torch.cat(refs), 2e-5 if dtype == torch.float32 else 2e-2, kernel)

    singles = [(0, p, 1) for p in (0, 1, 15, 16, 17, 32, 33, 63, 64, 100, 128, 299)] + [(1, 139, 1), (2, 6, 1)]
    portions = [(0, 0, 300), (1, 0, 2), (2, 0, 7), (1, 2, 131), (0, 171, 129), (1, 130, 10), (0, 64, 2)]
    run("general", singles + portions)
    pieces = dk % (4 if dtype == torch.float32 else 8) == 0 and dv % (4 if dtype == torch.float32 else 8) == 0
    assert ops.attention_span_decode_supported(dtype, dk, dv) == pieces
    if pieces:
        for ns in (1, 2, 5):
            run(ns, singles)
    assert ops.attention_span_prefill_supported(dtype, dk, dv) == (pieces and dtype == torch.bfloat16)
    if pieces and dtype == torch.bfloat16:
        run("prefill", portions + singles[:4])


# the requests' tokens cut into steps: whole portions, portions of two, single tokens beside portions, single tokens alone, a
# request left out of a step
LENS = [203, 40, 9]
STEPS = [[(0, 33), (1, 2), (2, 1)], [(1, 16), (0, 1)], [(2, 1), (0, 2), (1, 1)], [(0, 1), (1, 1), (2, 1)], [(1, 18)], [(2, 4), (0, 17)],
         [(0, 1), (2, 1)], [(0, 146), (1, 1)], [(1, 1), (0, 2), (2, 1)]]
SLOTS = [4, 1, 2]                                                  # of five; the others hold NaN


def _walk():
    """Per step: (token rows as (request, position), token_req, request starts, slots, single)."""
    at = [0] * len(LENS)
    for step in STEPS:
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


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H_,G,dk,dv,taps", [(4, 2, 24, 40, 4), (3, 1, 6, 9, 1), (2, 1, 128, 64, 5), (1, 1, 300, 200, 3), (6, 3, 32, 32, 2), (2, 2, 64, 136, 8)])
def test_delta_rule_with_one_decay_per_head(dtype, H_, G, dk, dv, taps):
    """Convolution, unit lengths, step sizes and decays, then the recurrence, over portions of unequal requests and single tokens
    in state slots with NaN around them; slow decays, the last query set to the first token's key."""
    from infinicore_infer_amd.kernels import ops
    g = torch.Generator().manual_seed(dk + taps)
    C = 2 * G * dk + H_ * dv
    x = [(2 * torch.randn(n, C + 2 * H_ + 5, generator=g)).to(dtype) for n in LENS]
    w = torch.randn(C, taps, generator=g) / math.sqrt(taps)
    rate, bias = torch.exp(torch.randn(H_, generator=g) - 3.0), torch.randn(H_, generator=g) - 2.0
    rows_want, beta_want, decay_want, o_want = [], [], [], []
    for r, n in enumerate(LENS):
        y = P.silu(P.short_conv(x[r][:, :C].double(), w.double()))
        qk = P.unit_length(y[:, :2 * G * dk].view(n, 2 * G, dk))
        beta = torch.sigmoid(x[r][:, C:C + H_].double())
        decay = torch.exp(-rate.double() * P.softplus(x[r][:, C + H_:C + 2 * H_].double() + bias.double()))
        q, k, v = qk[:, :G].repeat_interleave(H_ // G, 1), qk[:, G:].repeat_interleave(H_ // G, 1), y[:, 2 * G * dk:].view(n, H_, dv)
        q = q.clone()
        q[-1] = k[0]
        rows_want.append(torch.cat([qk.reshape(n, -1), y[:, 2 * G * dk:]], 1))
        beta_want.append(beta)
        decay_want.append(decay)
        o_want.append(P.delta_memory(q * dk ** -0.5, k, v, decay, beta).reshape(n, -1))
    pad, conv_at = 8, H_ * dk * dv
    st = torch.full((5, pad + conv_at + (taps - 1) * C), NAN, device="cuda")
    for s in SLOTS:
        st[s, pad:] = 0.0
    for rows, req, starts, slots, single in _walk():
        xx, T = _pick(x, rows).cuda(), len(rows)
        out, beta, decay = (torch.full((T, m), NAN, device="cuda") for m in (C, H_, H_))
        ops.delta_prep(xx[:, :C], w.cuda(), xx[:, C:C + H_], out, beta, G, H_, dk, dv, 1e-6, st, pad + conv_at, req, starts, slots, len(slots),
                       single, head_decay=(xx[:, C + H_:C + 2 * H_], rate.cuda(), bias.cuda(), decay))
        _close(out, _pick(rows_want, rows), 1e-5, "rows %s.." % (rows[0],))
        assert torch.allclose(beta.cpu().double(), _pick(beta_want, rows), atol=1e-6)
        assert torch.allclose(decay.cpu().double(), _pick(decay_want, rows), atol=1e-6)
        for t, (r, p) in enumerate(rows):
            if p == LENS[r] - 1:
                out[t, :G * dk] = rows_want[r][0, G * dk:2 * G * dk].float().cuda()
        for columns in ((None,) if single else (1, 2)):
            before = st.clone()
            o = torch.full((T, H_ * dv), NAN, device="cuda")
            ops.matrix_memory(out[:, :G * dk], out[:, G * dk:2 * G * dk], out[:, 2 * G * dk:], decay, H_, G, dk, dv, o, st, pad, starts, slots,
                              len(slots), single, scale=beta, delta=True, q_scale=dk ** -0.5, columns_a_thread=columns)
            _close(o, _pick(o_want, rows), 3e-5, "result %s.. columns %s" % (rows[0], columns))
            if columns == 1:
                st.copy_(before)
    assert bool(torch.isnan(st[0]).all()) and bool(torch.isnan(st[SLOTS][:, :pad]).all())


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("T,d", [(1, 96), (5, 70), (33, 1024), (3, 7000), (2, 3)])
@pytest.mark.parametrize("n", [1, 2, 3])
def test_results_added_to_the_stream_under_the_next_norm(dtype, T, d, n):
    from infinicore_infer_amd.kernels import ops
    g = torch.Generator().manual_seed(T + d)
    x = 3 * torch.randn(T, d, generator=g)
    w = 1 + 0.3 * torch.randn(d, generator=g)
    parts = [(torch.randn(T, d, generator=g).to(dtype), f) for f in (0.7, -1.3, 1.0)[:n]]
    want = x.double() + sum(f * y.double() for y, f in parts)
    for with_norm in (True, False):
        xs, out = x.cuda(), torch.full((T, d), NAN, dtype=dtype, device="cuda") if with_norm else None
        ops.branches_norm([(y.cuda(), f) for y, f in parts], w.cuda() if with_norm else None, xs, 1e-5, out=out)
        assert torch.allclose(xs.cpu().double(), want, atol=1e-5)
        if with_norm:
            _close(out, P.unit_rms(want, 1e-5) * w.double(), 1e-5 if dtype == torch.float32 else 1e-2, "norm")


@pytest.mark.parametrize("M,d,K", [(17, 256, 512), (64, 1024, 2048), (40, 2304, 640)])
@pytest.mark.parametrize("n", [0, 1, 2])
def test_sliced_products_take_other_results_along(M, d, K, n):
    from infinicore_infer_amd.kernels import ops
    g = torch.Generator().manual_seed(M + n)
    a, w = torch.randn(M, K, generator=g).to(torch.bfloat16), (torch.randn(d, K, generator=g) / math.sqrt(K)).to(torch.bfloat16)
    x, nw = torch.randn(M, d, generator=g), 1 + 0.3 * torch.randn(d, generator=g)
    also = [(torch.randn(M, d, generator=g).to(torch.bfloat16), f) for f in (0.6, -1.5)[:n]]
    slices = ops.gemm_splitk_slices(d, K)
    parts = ops.gemm_splitk(a.cuda(), w.cuda(), torch.empty(slices * M * d, device="cuda"), slices)
    xs, out = x.cuda(), torch.full((M, d), NAN, dtype=torch.bfloat16, device="cuda")
    ops.splitk_add_rmsnorm(parts, xs, 0.9, nw.cuda(), out, 1e-5, also=[(y.cuda(), f) for y, f in also])
    want = x.double() + 0.9 * (a.double() @ w.double().T) + sum(f * y.double() for y, f in also)
    assert torch.allclose(xs.cpu().double(), want, atol=2e-2)
    _close(out, P.unit_rms(want, 1e-5) * nw.double(), 1.5e-2, "norm")


# ---- generation through the entry point --------------------------------------------------------------------------------
def _plain_greedy(cfg, W, prompt, n):
    toks = list(prompt)
    for _ in range(n):
        toks.append(int(P.forward(cfg, W, toks, torch.float64)[-1].argmax()))
    return toks[len(prompt):]


@pytest.mark.parametrize("name", ["F1", "F2", "F3"])
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
    folder, W = _model(tmp_path_factory, "F2")
    prompt = H.random_tokens(F2["vocab"], 9, 77)
    r = subprocess.run([sys.executable, "-m", "infinicore_infer_amd.fokinex", "--amd", folder, "--dtype", "float32",
                        "--prompt-ids", ",".join(map(str, prompt)), "--max-new-tokens", "6", "--max-tokens", "128"],
                       cwd=H.__file__.rsplit("/tests/", 1)[0], capture_output=True, text=True, timeout=300)
    assert r.returncode == 0, r.stderr[-2000:]
    want = _plain_greedy(F2, W, prompt, 6)
    assert " ".join(map(str, want)) in " ".join(r.stdout.split()), r.stdout[-2000:]


def test_command_line_with_random_weights(tmp_path):
    import subprocess
    import sys
    path = str(tmp_path / "config.json")
    with open(path, "w") as f:
        json.dump(F3, f)
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
    folder, W = _model(tmp_path_factory, "F1")
    requests = _requests("F1", seed=4)
    steps, max_tokens = H.trace_mixed(requests, seed=3)
    root = H.__file__.rsplit("/tests/", 1)[0]
    out = str(tmp_path / "out")
    r = subprocess.run([os.path.join(root, "bin", "trace_run"), "--model", folder, "--dtype", "float32", "--out", out,
                        "--max-tokens", str(max_tokens)], input="\n".join(json.dumps(s) for s in steps) + "\n",
                       capture_output=True, text=True, timeout=300, cwd=root)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [l for l in r.stdout.split("\n") if l.startswith("done")] == ["done %d" % s["step"] for s in steps]
    ref = {rid: P.forward(F1, W, toks, torch.float64) for rid, toks in requests.items()}
    at, got = {}, {}
    for s in steps:
        rows = torch.frombuffer(bytearray(open(os.path.join(out, "%d.f32" % s["step"]), "rb").read()), dtype=torch.float32).view(-1, F1["vocab"])
        i = 0
        for e in s["entries"]:
            for w in e["want"]:
                got[(e["id"], at.get(e["id"], 0) + w)] = rows[i].clone()
                i += 1
            at[e["id"]] = at.get(e["id"], 0) + len(e["tokens"])
        assert i == rows.shape[0]
    H.compare(got, ref, 1e-4, "trace runner", steps)


# ---- configurations drawn from seeds -------------------------------------------------------------------------------------
def _drawn_config(seed):
    rng = random.Random(seed)
    layers, sources = [], []
    ff = lambda: None if rng.random() < 0.2 else rng.choice([12, 30, 64, 96])
    window = lambda: rng.choice([None, 1, 2, 9, 16, 33, 64, 100])
    for i in range(rng.choice([2, 3, 4, 5])):
        if rng.random() < 0.4:
            kv, dim = rng.choice([1, 2, 3]), rng.choice([8, 12, 32, 48, 64, 96])
            kv2 = rng.choice([1, 2, 3])
            layers.append(_parallel((kv * rng.choice([1, 2, 4]), kv, dim, round(rng.uniform(0.05, 0.5), 3), rng.choice([1.5, 10.0, 50.0]), window()),
                                    (kv2 * rng.choice([1, 2, 3]), kv2, rng.choice([4, 12, 32, 50]), rng.choice([5, 16, 33, 64]), rng.choice([1, 2, 3, 4, 6])),
                                    (round(rng.uniform(0.4, 1.5), 2), round(rng.uniform(0.4, 1.5), 2)), ff()))
            continue
        own = not sources or rng.random() < 0.5
        if own:
            kv_rank, rot_dim = rng.choice([16, 22, 64, 96, 128]), rng.choice([2, 8, 16, 32])
            rot = (rng.choice([100.0, 10000.0, 3e5]), rng.choice([None, (2.0, 16, 4.0, 0.5), (8.0, 128, 32.0, 1.0), (40.0, 4096, 32.0, 1.0)]))
            sources.append((i, kv_rank, rot_dim, rot))
        j, kv_rank, rot_dim, rot = sources[-1] if own else rng.choice(sources)
        layers.append(_latent(rng.choice([1, 2, 5, 8]), rng.choice([8, 10, 32, 64]), rot_dim, rng.choice([8, 14, 40, 64, 96]), rng.choice([8, 20, 48]),
                              kv_rank, round(rng.uniform(0.08, 0.4), 3), window(), rot, None if own else j, ff()))
    return {"architecture": "Fokinex", "vocab": rng.choice([53, 128, 301]), "width": rng.choice([34, 48, 64, 100]),
            "norm": {"eps": rng.choice([1e-5, 1e-6, 1e-3])}, "embedding": {"scale": rng.choice([0.3, 1.0, 12.0])}, "layers": layers}


@pytest.mark.parametrize("seed", list(range(14)))
def test_drawn_configurations(tmp_path_factory, seed):
    from infinicore_infer_amd.engine import Engine
    cfg = _drawn_config(seed)
    folder = os.path.join(str(tmp_path_factory.getbasetemp()), "fokinex_drawn_%d" % seed)
    W = _write_model(folder, cfg, seed)
    rng = random.Random(seed + 100)
    requests = {"r%d" % i: H.random_tokens(cfg["vocab"], n, seed * 10 + i)
                for i, n in enumerate([rng.choice([1, 2, 5, 40, 66, 129, 150]) for _ in range(5)])}
    ref = {rid: P.forward(cfg, W, toks, torch.float64) for rid, toks in requests.items()}
    steps, max_tokens = H.trace_mixed(requests, sizes=(7, 2, 40, 3, 11, 2, 70, 33), seed=seed)
    for dname, dtype, tol in DTYPES:
        engine = Engine.from_dir(folder, dtype=dtype, max_tokens=max_tokens, page_size=16, max_requests=4)
        if dtype == torch.bfloat16:
            tol = _bf16_tolerance(cfg, W, requests, ref)
        worst = H.compare(H.run_trace(engine, steps), ref, tol, "drawn %d %s" % (seed, dname), steps)
        print("drawn %d %s: worst error %.3g (allowed %.3g)" % (seed, dname, worst[0], tol))
        engine.cache.check_invariants()
        assert not engine.cache.requests
