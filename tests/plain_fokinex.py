"""A plain, slow implementation of the Fokinex decoder, written from its equations for the tests.

One function per mechanism, whole sequences at once, keys and values made for every head, dense scores, a loop over tokens
for the recurrence, no cache, no kernels and no code of the package.  Everything runs in one dtype (float64 by default).

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


# ---- which keys a query sees ------------------------------------------------------------------------------
def seen_keys(T, window):
    """[T, T] bool: query i sees key j when 0 <= i - j < window (no window: every j <= i)."""
    back = torch.arange(T)[:, None] - torch.arange(T)[None, :]
    return (back >= 0) & (back < window) if window else back >= 0


# ---- rotation with stretched wavelengths ------------------------------------------------------------------
def stretched_frequencies(dims, base, scaling=None):
    """(frequencies, factor on cos and sin): base^(-2i/dims), slow ones divided by ``factor``, fast ones as they are, a ramp
    over the pair index between the two."""
    f = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    if not scaling:
        return f, 1.0
    factor, original = scaling["factor"], scaling["original"]
    index_of = lambda turns: dims * math.log(original / (2 * math.pi * turns)) / (2 * math.log(base))
    lo, hi = max(math.floor(index_of(scaling["fast"])), 0), min(math.ceil(index_of(scaling["slow"])), dims - 1)
    out = []
    for i, v in enumerate(f):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(v / factor * ramp + v * (1.0 - ramp))
    return out, 0.1 * math.log(factor) + 1.0


def rotate_pairs(x, positions, rot):
    """x [T, .., size]: entries (2i, 2i + 1) of the first rot.dims turn together; the rest stay."""
    dims = rot["dims"]
    freq, mult = stretched_frequencies(dims, rot["base"], rot.get("scaling"))
    out = x.clone()
    for i in range(dims // 2):
        a = torch.as_tensor([pos * freq[i] for pos in positions], dtype=x.dtype).view(-1, *([1] * (x.dim() - 2)))
        c, s = torch.cos(a) * mult, torch.sin(a) * mult
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        out[..., 2 * i] = u * c - v * s
        out[..., 2 * i + 1] = v * c + u * s
    return out


def softmax_with_sink(s, sink=None):
    """Softmax over the last axis; ``sink``: a number whose exponential joins the denominator."""
    m = s.max(-1, keepdim=True).values
    if sink is not None:
        m = torch.maximum(m, sink)
    e = torch.exp(s - m)
    den = e.sum(-1, keepdim=True)
    if sink is not None:
        den = den + torch.exp(sink - m)
    return e / den


# ---- attention through a latent ---------------------------------------------------------------------------
def latent_rows(h, W, p, m, eps):
    """What a layer caches: (the normed latent [T, kv_rank], the rotated key part [T, rot_dim])."""
    rows = h @ W[p + "dkv"].T
    R = m["kv_rank"]
    return unit_rms(rows[:, :R], eps) * W[p + "dkv.norm"], rotate_pairs(rows[:, R:], range(h.shape[0]), m["rot"])


def latent_attention(h, W, p, m, eps, rows):
    """``rows``: the latent and the rotated key part this layer reads (its own, or another layer's)."""
    T, H, dim, E, dv = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    c, k_rot = rows
    q = (unit_rms(h @ W[p + "dq"].T, eps) * W[p + "dq.norm"]) @ W[p + "uq"].T
    q = q.reshape(T, H, dim + E)
    q_rot = rotate_pairs(q[..., dim:], range(T), m["rot"])
    k, v = (c @ W[p + "uk"].T).reshape(T, H, dim), (c @ W[p + "uv"].T).reshape(T, H, dv)
    seen = seen_keys(T, (m.get("mask") or {}).get("size"))
    out = []
    for hd in range(H):
        s = (q[:, hd, :dim] @ k[:, hd].T + q_rot[:, hd] @ k_rot.T) * m["scale"]
        out.append(softmax_with_sink(s.masked_fill(~seen, -math.inf), W[p + "sink"][hd]) @ v[:, hd])
    return torch.cat(out, -1) @ W[p + "o"].T


# ---- attention whose values are its keys ------------------------------------------------------------------
def tied_attention(h, W, p, m, eps):
    """Values are the projected keys before their norm; norms over whole rows; capped scores with a slope per head over the
    distance taken off; a gate on the heads."""
    T, H, dim = h.shape[0], m["heads"], m["dim"]
    G = m.get("kv_heads") or H
    k_raw = h @ W[p + "k"].T
    q = (unit_rms(h @ W[p + "q"].T, eps) * W[p + "q.norm"]).reshape(T, H, dim)
    k = (unit_rms(k_raw, eps) * W[p + "k.norm"]).reshape(T, G, dim)
    v = k_raw.reshape(T, G, dim)
    seen = seen_keys(T, (m.get("mask") or {}).get("size"))
    back = (torch.arange(T)[:, None] - torch.arange(T)[None, :]).to(h.dtype)
    out = []
    for hd in range(H):
        g = hd // (H // G)
        s = (q[:, hd] @ k[:, g].T) * m["scale"]
        s = m["softcap"] * torch.tanh(s / m["softcap"])
        s = s - 2.0 ** (-8.0 * (hd + 1) / H) * back
        out.append(softmax_with_sink(s.masked_fill(~seen, -math.inf)) @ v[:, g])
    return (torch.cat(out, -1) * torch.sigmoid(h @ W[p + "g"].T)) @ W[p + "o"].T


# ---- delta rule with one decay per head -------------------------------------------------------------------
def short_conv(x, w):
    """x [T, C], w [C, taps]; the last column multiplies the current token, zeros stand before the start."""
    T, C = x.shape
    taps = w.shape[1]
    padded = torch.cat([torch.zeros(taps - 1, C, dtype=x.dtype), x], dim=0)
    out = torch.zeros_like(x)
    for j in range(taps):
        out = out + w[:, j] * padded[j:j + T]
    return out


def delta_memory(q, k, v, decay, beta):
    """S <- decay * S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q; q, k [T, heads, dim], decay, beta [T, heads]."""
    T, heads, dim = q.shape
    S = torch.zeros(heads, dim, v.shape[2], dtype=q.dtype)
    out = torch.zeros(T, heads, v.shape[2], dtype=q.dtype)
    for t in range(T):
        S = decay[t][:, None, None] * S
        u = beta[t][:, None] * (v[t] - (S * k[t][:, :, None]).sum(1))
        S = S + k[t][:, :, None] * u[:, None, :]
        out[t] = (S * q[t][:, :, None]).sum(1)
    return out


def delta_mixer(h, W, p, m, eps):
    T, H, dim, dv = h.shape[0], m["heads"], m["dim"], m["vdim"]
    G = m.get("kv_heads") or H
    q, k, v = (silu(short_conv(h @ W[p + n].T, W[p + n + ".conv"])) for n in ("q", "k", "v"))
    q = unit_length(q.reshape(T, G, dim)).repeat_interleave(H // G, 1) * dim ** -0.5
    k = unit_length(k.reshape(T, G, dim)).repeat_interleave(H // G, 1)
    beta = torch.sigmoid(h @ W[p + "b"].T)
    decay = torch.exp(-torch.exp(W[p + "A_log"]) * softplus(h @ W[p + "a"].T + W[p + "dt_bias"]))
    o = unit_rms(delta_memory(q, k, v.reshape(T, H, dv), decay, beta), eps) * W[p + "norm"]
    return (o.reshape(T, H * dv) * silu(h @ W[p + "g"].T)) @ W[p + "o"].T


def parallel_mixer(h, W, p, m, eps):
    return (m["left_scale"] * tied_attention(h, W, p + "left.", m["left"], eps)
            + m["right_scale"] * delta_mixer(h, W, p + "right.", m["right"], eps))


# ---- feed-forward and the model ---------------------------------------------------------------------------
def gated_unit(h, W, p):
    return (silu(h @ W[p + "gate"].T) * (h @ W[p + "up"].T)) @ W[p + "down"].T


def forward(cfg, W, tokens, dtype=torch.float64, layers_out=None, rnd=lambda x: x):
    """Logits [T, vocab] of one whole sequence.  ``layers_out``: a list that receives the residual stream after every layer.
    ``rnd``: applied to what every sublayer reads and returns (a rounding shows how far rounding alone moves the logits)."""
    W = {k: v.to(dtype) for k, v in W.items()}
    eps = cfg["norm"]["eps"]
    x = W["embed"][torch.as_tensor(list(tokens), dtype=torch.long)] * (cfg.get("embedding") or {}).get("scale", 1.0)
    kept = {}
    for i, l in enumerate(cfg["layers"]):
        p, m = "l%d." % i, l["mixer"]
        h = rnd(unit_rms(x, eps) * W[p + "norm1"])
        if l["type"] == "latent_attention":
            if m.get("kv_from") is None:
                kept[i] = tuple(rnd(z) for z in latent_rows(h, W, p + "mix.", m, eps))
            y = latent_attention(h, W, p + "mix.", m, eps, kept[i if m.get("kv_from") is None else m["kv_from"]])
        elif l["type"] == "parallel":
            y = parallel_mixer(h, W, p + "mix.", m, eps)
        else:
            raise ValueError(l["type"])
        y = rnd(y)
        if l.get("mlp"):
            y = y + rnd(gated_unit(h, W, p + "mlp."))
        x = x + y
        if layers_out is not None:
            layers_out.append(x.clone())
    return rnd(unit_rms(x, eps) * W["final.norm"]) @ W["head"].T


# ---- random weights for the tests -------------------------------------------------------------------------
def random_weights(cfg, seed):
    """Every tensor of a configuration, float32 values that bfloat16 holds exactly."""
    g = torch.Generator().manual_seed(seed)
    d = cfg["width"]
    lin = lambda o, i, s=1.0: torch.randn(o, i, generator=g) * (s / math.sqrt(i))
    around = lambda n, mean=0.0, s=0.2: mean + s * torch.randn(n, generator=g)
    conv = lambda c, taps: torch.randn(c, taps, generator=g) / math.sqrt(taps)
    scale = (cfg.get("embedding") or {}).get("scale", 1.0)
    W = {"embed": torch.randn(cfg["vocab"], d, generator=g) / scale, "head": lin(cfg["vocab"], d, 2.0), "final.norm": around(d, 1.0)}

    def latent(p, m):
        H, R, E, q = m["heads"], m["kv_rank"], m["rot_dim"], m["q_rank"]
        W[p + "dq"], W[p + "dq.norm"] = lin(q, d), around(q, 1.0)
        W[p + "uq"] = lin(H * (m["dim"] + E), q, 2.0)
        if m.get("kv_from") is None:
            W[p + "dkv"], W[p + "dkv.norm"] = lin(R + E, d), around(R, 1.0)
        W[p + "uk"], W[p + "uv"] = lin(H * m["dim"], R, 1.5), lin(H * m["vdim"], R)
        W[p + "sink"], W[p + "o"] = around(H, 0.5, 1.0), lin(d, H * m["vdim"], 2.0)

    def tied(p, m):
        H, G, dk = m["heads"], m.get("kv_heads") or m["heads"], m["dim"]
        W[p + "q"], W[p + "k"], W[p + "g"] = lin(H * dk, d), lin(G * dk, d), lin(H * dk, d, 2.0)
        W[p + "q.norm"], W[p + "k.norm"] = around(H * dk, 1.3), around(G * dk, 1.3)
        W[p + "o"] = lin(d, H * dk, 3.0)

    def delta(p, m):
        H, G, dk, dv = m["heads"], m.get("kv_heads") or m["heads"], m["dim"], m["vdim"]
        for n, c in (("q", G * dk), ("k", G * dk), ("v", H * dv)):
            W[p + n], W[p + n + ".conv"] = lin(c, d, 2.0), conv(c, m["conv"])
        W[p + "b"], W[p + "A_log"], W[p + "a"], W[p + "dt_bias"] = lin(H, d, 2.0), around(H, -1.0, 1.0), lin(H, d, 2.0), around(H, -2.0, 1.5)
        W[p + "norm"], W[p + "g"], W[p + "o"] = around(dv, 1.0), lin(H * dv, d, 2.0), lin(d, H * dv, 2.0)

    for i, l in enumerate(cfg["layers"]):
        p, m = "l%d." % i, l["mixer"]
        W[p + "norm1"] = around(d, 1.0)
        if l["type"] == "latent_attention":
            latent(p + "mix.", m)
        else:
            tied(p + "mix.left.", m["left"])
            delta(p + "mix.right.", m["right"])
        if l.get("mlp"):
            ff = l["mlp"]["ff"]
            W[p + "mlp.gate"], W[p + "mlp.up"], W[p + "mlp.down"] = lin(ff, d, 2.0), lin(ff, d), lin(d, ff)
    return {k: v.to(torch.bfloat16).to(torch.float32) for k, v in W.items()}
