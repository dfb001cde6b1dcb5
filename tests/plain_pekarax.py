"""A plain, slow implementation of the Pekarax decoder, written from its equations for the tests.

One function per mechanism, whole sequences at once, a loop over tokens for every recurrence and over tokens and experts
for the routing, no cache, no kernels and no code of the package.  Everything runs in one dtype (float64 by default).

Notation: T tokens, d the residual width, W a dict name -> tensor, linear weights [out, in], p a tensor prefix,
r(z) = z / sqrt(mean(z^2) + eps) over the last axis.
"""
import math

import torch


def unit_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def unit_length(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def silu(z):
    return z * torch.sigmoid(z)


def softplus(z):
    return torch.log1p(torch.exp(-z.abs())) + torch.clamp(z, min=0.0)


# ---- short causal convolution -----------------------------------------------------------------------------
def short_conv(x, w):
    """x [T, C], w [C, taps]; the last column multiplies the current token, zeros stand before the start."""
    T, C = x.shape
    taps = w.shape[1]
    padded = torch.cat([torch.zeros(taps - 1, C, dtype=x.dtype), x], dim=0)
    out = torch.zeros_like(x)
    for j in range(taps):
        out = out + w[:, j] * padded[j:j + T]
    return out


# ---- rotation of halves -----------------------------------------------------------------------------------
def rotate_halves(x, positions, dims, base):
    """x [T, heads, size]: entry i < dims/2 turns with entry i + dims/2 by position * base^(-2i/dims); the rest stay."""
    out = x.clone()
    h = dims // 2
    for i in range(h):
        a = torch.as_tensor([pos * base ** (-2.0 * i / dims) for pos in positions], dtype=x.dtype)[:, None]
        c, s = torch.cos(a), torch.sin(a)
        u, v = x[..., i], x[..., i + h]
        out[..., i] = u * c - v * s
        out[..., i + h] = v * c + u * s
    return out


# ---- softmax attention over every earlier token -----------------------------------------------------------
def conv_attention(h, W, p, heads, kv_heads, dim, vdim, scale, rot_dims, rot_base, eps):
    """q, k, v through a convolution each, q and k rotated, then brought to unit root mean square per head."""
    T = h.shape[0]
    q, k, v = h @ W[p + "q"].T, h @ W[p + "k"].T, h @ W[p + "v"].T
    if p + "q.conv" in W:
        q, k, v = (short_conv(z, W[p + n + ".conv"]) for z, n in ((q, "q"), (k, "k"), (v, "v")))
    q, k, v = q.reshape(T, heads, dim), k.reshape(T, kv_heads, dim), v.reshape(T, kv_heads, vdim)
    if rot_dims:
        q, k = rotate_halves(q, range(T), rot_dims, rot_base), rotate_halves(k, range(T), rot_dims, rot_base)
    q, k = unit_rms(q, eps), unit_rms(k, eps)
    seen = torch.tril(torch.ones(T, T, dtype=torch.bool))
    out = []
    for hd in range(heads):
        g = hd // (heads // kv_heads)
        s = ((q[:, hd] @ k[:, g].T) * scale).masked_fill(~seen, -math.inf)
        out.append(torch.softmax(s, -1) @ v[:, g])
    return torch.cat(out, -1) @ W[p + "o"].T


# ---- matrix memory with exponential gates -----------------------------------------------------------------
def matrix_memory(q, k, v, log_i, log_f):
    """q, k [T, heads, dim], v [T, heads, vdim], log gates [T, heads]; S, n and the running maximum start at zero."""
    T, heads, dim = q.shape
    S = torch.zeros(heads, dim, v.shape[2], dtype=q.dtype)
    n = torch.zeros(heads, dim, dtype=q.dtype)
    m = torch.zeros(heads, dtype=q.dtype)
    out = torch.zeros(T, heads, v.shape[2], dtype=q.dtype)
    for t in range(T):
        m_new = torch.maximum(log_f[t] + m, log_i[t])
        keep, add = torch.exp(log_f[t] + m - m_new), torch.exp(log_i[t] - m_new)
        S = keep[:, None, None] * S + add[:, None, None] * k[t][:, :, None] * v[t][:, None, :]
        n = keep[:, None] * n + add[:, None] * k[t]
        m = m_new
        den = torch.maximum((n * q[t]).sum(-1).abs(), torch.exp(-m)) + 1e-6
        out[t] = (S * q[t][:, :, None]).sum(1) / den[:, None]
    return out


def mlstm_mixer(h, W, p, heads, dim, vdim, cap, eps):
    T = h.shape[0]
    q = (h @ W[p + "q"].T).reshape(T, heads, dim) * dim ** -0.5
    k = (h @ W[p + "k"].T).reshape(T, heads, dim)
    v = (h @ W[p + "v"].T).reshape(T, heads, vdim)
    log_i = cap * torch.tanh((h @ W[p + "i"].T + W[p + "i.b"]) / cap)
    log_f = -softplus(-cap * torch.tanh((h @ W[p + "f"].T + W[p + "f.b"]) / cap))
    o = unit_rms(matrix_memory(q, k, v, log_i, log_f), eps).reshape(T, heads * vdim)
    return (o * W[p + "norm"] * torch.sigmoid(h @ W[p + "g"].T)) @ W[p + "o"].T


def parallel_mixer(h, W, p, m, eps):
    l, r = m["left"], m["right"]
    rot = l.get("rot") or {}
    left = conv_attention(h, W, p + "left.", l["heads"], l.get("kv_heads") or l["heads"], l["dim"], l.get("vdim") or l["dim"], l["scale"],
                          rot.get("dims") or 0, rot.get("base") or 10000.0, eps)
    right = mlstm_mixer(h, W, p + "right.", r["heads"], r["dim"], r["vdim"], r["gate_cap"], eps)
    return m["left_scale"] * left + m["right_scale"] * right


# ---- gated linear attention with a decay per key channel --------------------------------------------------
def channel_decay_memory(q, k, v, decay):
    """S <- diag(decay) S + k v^T, o = S^T q; q, k, decay [T, heads, dim], v [T, heads, vdim]."""
    T, heads, dim = q.shape
    S = torch.zeros(heads, dim, v.shape[2], dtype=q.dtype)
    out = torch.zeros(T, heads, v.shape[2], dtype=q.dtype)
    for t in range(T):
        S = decay[t][:, :, None] * S + k[t][:, :, None] * v[t][:, None, :]
        out[t] = (S * q[t][:, :, None]).sum(1)
    return out


def gla_mixer(h, W, p, heads, dim, vdim, tau, eps):
    T = h.shape[0]
    q = (h @ W[p + "q"].T).reshape(T, heads, dim) * dim ** -0.5
    k = (h @ W[p + "k"].T).reshape(T, heads, dim)
    v = (h @ W[p + "v"].T).reshape(T, heads, vdim)
    z = (h @ W[p + "a1"].T) @ W[p + "a2"].T + W[p + "a2.b"]
    decay = torch.exp(-softplus(-z) / tau).reshape(T, heads, dim)
    o = unit_rms(channel_decay_memory(q, k, v, decay), eps) * W[p + "norm"]
    return (o.reshape(T, heads * vdim) * silu(h @ W[p + "g"].T)) @ W[p + "o"].T


# ---- delta rule with a decay per key channel --------------------------------------------------------------
def delta_memory(q, k, v, decay, beta):
    """S <- decay * S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q; q, k, decay [T, heads, dim], beta [T, heads]."""
    T, heads, dim = q.shape
    S = torch.zeros(heads, dim, v.shape[2], dtype=q.dtype)
    out = torch.zeros(T, heads, v.shape[2], dtype=q.dtype)
    for t in range(T):
        S = decay[t][:, :, None] * S
        u = beta[t][:, None] * (v[t] - (S * k[t][:, :, None]).sum(1))
        S = S + k[t][:, :, None] * u[:, None, :]
        out[t] = (S * q[t][:, :, None]).sum(1)
    return out


def channel_delta_mixer(h, W, p, heads, kv_heads, dim, vdim, eps):
    T = h.shape[0]
    q, k, v = (silu(short_conv(h @ W[p + n].T, W[p + n + ".conv"])) for n in ("q", "k", "v"))
    per = heads // kv_heads
    q = unit_length(q.reshape(T, kv_heads, dim)).repeat_interleave(per, 1) * dim ** -0.5
    k = unit_length(k.reshape(T, kv_heads, dim)).repeat_interleave(per, 1)
    v = v.reshape(T, heads, vdim)
    beta = torch.sigmoid(h @ W[p + "b"].T)
    step = softplus((h @ W[p + "a1"].T) @ W[p + "a2"].T + W[p + "dt_bias"]).reshape(T, heads, dim)
    decay = torch.exp(-torch.exp(W[p + "A_log"])[None, :, None] * step)
    o = unit_rms(delta_memory(q, k, v, decay, beta), eps) * W[p + "norm"]
    gate = torch.sigmoid((h @ W[p + "g1"].T) @ W[p + "g2"].T)
    return (o.reshape(T, heads * vdim) * gate) @ W[p + "o"].T


# ---- feed-forward -----------------------------------------------------------------------------------------
def bounded_unit(h, W, p, limit):
    g = torch.clamp(h @ W[p + "gate"].T, max=limit)
    u = torch.clamp(h @ W[p + "up"].T, -limit, limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1.0)) @ W[p + "down"].T


def choose(s, correction, top, groups, keep):
    """The ``top`` places with the largest corrected scores among the ``keep`` best of ``groups`` equal runs of neighbours
    (a run is as good as its best corrected score); the lower place wins a tie."""
    c = [float(a) for a in s + correction]
    size = len(c) // groups
    best = [max(c[g * size:(g + 1) * size]) for g in range(groups)]
    kept = sorted(range(groups), key=lambda g: (-best[g], g))[:keep]
    return sorted((e for e in range(len(c)) if e // size in kept), key=lambda e: (-c[e], e))[:top]


def routed_experts(h, W, p, mlp):
    r = mlp["router"]
    experts, identity = r["experts"], r.get("identity") or 0
    groups = r.get("groups") or {"count": 1, "keep": 1}
    s = torch.softmax(h @ W[p + "router"].T, -1)
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        chosen = choose(s[t], W[p + "correction"], r["top"], groups["count"], groups["keep"])
        total = sum(s[t, e] for e in chosen) + 1e-20
        for e in chosen:
            y = bounded_unit(h[t][None], W, "%se%d." % (p, e), mlp["expert"]["limit"])[0] if e < experts else h[t]
            out[t] = out[t] + s[t, e] / total * r.get("scale", 1.0) * y
    assert s.shape[1] == experts + identity
    return out


# ---- the model --------------------------------------------------------------------------------------------
def run_mixer(h, W, p, kind, m, eps):
    if kind == "parallel":
        return parallel_mixer(h, W, p, m, eps)
    if kind == "gla":
        return gla_mixer(h, W, p, m["heads"], m["dim"], m["vdim"], m["tau"], eps)
    if kind == "channel_delta":
        return channel_delta_mixer(h, W, p, m["heads"], m.get("kv_heads") or m["heads"], m["dim"], m["vdim"], eps)
    raise ValueError(kind)


def sum_then_norm(x, y, w, alpha, eps):
    """The norm sits after the residual sum: r(alpha x + y) (1 + w)."""
    return unit_rms(alpha * x + y, eps) * (1.0 + w)


def forward(cfg, W, tokens, dtype=torch.float64, layers_out=None, rnd=lambda x: x):
    """Logits [T, vocab] of one whole sequence.  ``layers_out``: a list that receives the residual stream after every layer.
    ``rnd``: applied to what every sublayer reads and returns (a rounding shows how far rounding alone moves the logits)."""
    W = {k: (v.to(dtype) if v.is_floating_point() else v) for k, v in W.items()}
    eps, alpha = cfg["norm"]["eps"], cfg["postln_alpha"]
    x = W["embed"][torch.as_tensor(list(tokens), dtype=torch.long)]
    for i, l in enumerate(cfg["layers"]):
        p = "l%d." % i
        x = sum_then_norm(x, rnd(run_mixer(rnd(x), W, p + "mix.", l["type"], l["mixer"], eps)), W[p + "norm1"], alpha, eps)
        if l.get("mlp"):
            x = sum_then_norm(x, rnd(routed_experts(rnd(x), W, p + "mlp.", l["mlp"])), W[p + "norm2"], alpha, eps)
        if layers_out is not None:
            layers_out.append(x.clone())
    return rnd(unit_rms(x, eps) * (1.0 + W["final.norm"])) @ W["head"].T


# ---- random weights for the tests -------------------------------------------------------------------------
def random_weights(cfg, seed, ranks=(12, 20)):
    """Every tensor of a configuration, float32 values that bfloat16 holds exactly.  ``ranks``: the inner sizes of the
    low-rank products (decays, output gates)."""
    g = torch.Generator().manual_seed(seed)
    d = cfg["width"]
    lin = lambda o, i, s=1.0: torch.randn(o, i, generator=g) * (s / math.sqrt(i))
    around = lambda n, mean=0.0, s=0.2: mean + s * torch.randn(n, generator=g)
    conv = lambda c, taps: torch.randn(c, taps, generator=g) / math.sqrt(taps)
    W = {"embed": torch.randn(cfg["vocab"], d, generator=g), "head": lin(cfg["vocab"], d, 2.0), "final.norm": around(d)}

    def delta(p, m):
        H, G, dk, dv = m["heads"], m.get("kv_heads") or m["heads"], m["dim"], m["vdim"]
        for n, c in (("q", G * dk), ("k", G * dk), ("v", H * dv)):
            W[p + n], W[p + n + ".conv"] = lin(c, d, 2.0), conv(c, m["conv"])
        W[p + "b"], W[p + "A_log"] = lin(H, d, 2.0), around(H, -1.0, 1.0)
        W[p + "a1"], W[p + "a2"], W[p + "dt_bias"] = lin(ranks[0], d), lin(H * dk, ranks[0], 2.0), around(H * dk, -2.0, 1.5)
        W[p + "g1"], W[p + "g2"] = lin(ranks[1], d, 2.0), lin(H * dv, ranks[1])
        W[p + "norm"], W[p + "o"] = around(dv, 1.0), lin(d, H * dv, 2.0)

    def gla(p, m):
        H, dk, dv = m["heads"], m["dim"], m["vdim"]
        W[p + "q"], W[p + "k"], W[p + "v"], W[p + "g"] = lin(H * dk, d, 2.0), lin(H * dk, d), lin(H * dv, d), lin(H * dv, d, 2.0)
        W[p + "a1"], W[p + "a2"], W[p + "a2.b"] = lin(ranks[0], d), lin(H * dk, ranks[0], 2.0), around(H * dk, 1.0, 2.0)
        W[p + "norm"], W[p + "o"] = around(dv, 1.0), lin(d, H * dv, 2.0)

    def attention(p, m):
        H, G = m["heads"], m.get("kv_heads") or m["heads"]
        dk, dv = m["dim"], m.get("vdim") or m["dim"]
        for n, c in (("q", H * dk), ("k", G * dk), ("v", G * dv)):
            W[p + n] = lin(c, d)
            if m.get("conv"):
                W[p + n + ".conv"] = conv(c, m["conv"])
        W[p + "o"] = lin(d, H * dv)

    def mlstm(p, m):
        H, dk, dv = m["heads"], m["dim"], m["vdim"]
        W[p + "q"], W[p + "k"], W[p + "v"], W[p + "g"] = lin(H * dk, d, 2.0), lin(H * dk, d), lin(H * dv, d), lin(H * dv, d, 2.0)
        W[p + "i"], W[p + "i.b"], W[p + "f"], W[p + "f.b"] = lin(H, d, 3.0), around(H, -1.0, 1.0), lin(H, d, 2.0), around(H, 3.0, 1.0)
        W[p + "norm"], W[p + "o"] = around(H * dv, 1.0), lin(d, H * dv)

    for i, l in enumerate(cfg["layers"]):
        p, m = "l%d." % i, l["mixer"]
        W[p + "norm1"] = around(d)
        if l["type"] == "channel_delta":
            delta(p + "mix.", m)
        elif l["type"] == "gla":
            gla(p + "mix.", m)
        else:
            attention(p + "mix.left.", m["left"])
            mlstm(p + "mix.right.", m["right"])
        if l.get("mlp"):
            r, ff = l["mlp"]["router"], l["mlp"]["expert"]["ff"]
            W[p + "norm2"] = around(d)
            for e in range(r["experts"]):
                q = "%smlp.e%d." % (p, e)
                W[q + "gate"], W[q + "up"], W[q + "down"] = lin(ff, d, 2.0), lin(ff, d), lin(d, ff)
            total = r["experts"] + (r.get("identity") or 0)
            W[p + "mlp.router"], W[p + "mlp.correction"] = lin(total, d, 2.0), around(total, 0.0, 0.15)
    return {k: v.to(torch.bfloat16).to(torch.float32) for k, v in W.items()}
