"""Plain, slow implementation of the Pitelorn design, written from its equations: one
function per mechanism, whole sequences at a time, no cache, no package code.

A model is (cfg, tensors): ``cfg`` the parsed ``config.json`` dict, ``tensors`` a dict of
torch tensors by checkpoint name.  Everything is evaluated in ``DT`` (float64 by default,
so that the comparison's error is the framework's alone).

Notation: T tokens, x the residual [T, width], t = 0..T-1 the positions.
"""
import math

import torch

DT = torch.float64


def _t(x):
    return x.to(DT)


def lin(ten, name, h):
    return h @ _t(ten[name]).T


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def offset_norm(x, w, eps):
    """Residual-stream norm: the stored weight is an offset from one."""
    return rms(x, eps) * (1.0 + _t(w))


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return torch.log1p(torch.exp(-z.abs())) + z.clamp_min(0.0)


# ------------------------------------------------------------------------------ embedding
def embedding(cfg, ten, tokens):
    """Token row plus a row of the pair table chosen by the previous and the current token."""
    x = _t(ten["embed"])[list(tokens)]
    pair = (cfg.get("embedding") or {}).get("bigram")
    if pair:
        n = pair["buckets"]
        rows = [n] + [(a * pair["mul_prev"] + b * pair["mul_cur"]) % n for a, b in zip(tokens[:-1], tokens[1:])]
        x = x + _t(ten["bigram"])[rows[:len(tokens)]]
    return x


# ------------------------------------------------------------------------------ positions
def frequencies(rot):
    """Per pair the angle per position, and the factor on cos and sin."""
    dims, base = rot["dims"], float(rot["base"])
    f = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    sc = rot.get("scaling")
    if not sc:
        return f, 1.0
    s, orig = float(sc["factor"]), float(sc["original"])

    def pair_of(turns):
        return dims * math.log(orig / (2.0 * math.pi * turns)) / (2.0 * math.log(base))

    lo = max(math.floor(pair_of(sc["fast"])), 0)
    hi = min(math.ceil(pair_of(sc["slow"])), dims - 1)
    out = []
    for i, fi in enumerate(f):
        r = (i - lo) / max(hi - lo, 0.001)
        r = 0.0 if r < 0.0 else 1.0 if r > 1.0 else r
        out.append(fi / s * r + fi * (1.0 - r))
    return out, 0.1 * math.log(s) + 1.0


def rotate(x, rot, neighbours):
    """x [T, heads, dim]: pairs (2i, 2i + 1) if ``neighbours``, else (i, i + dims/2), of the
    first dims entries of every head."""
    if not rot or not rot.get("dims"):
        return x
    dims = rot["dims"]
    f, mult = frequencies(rot)
    out = x.clone()
    for t in range(x.shape[0]):
        for i, fi in enumerate(f):
            a, b = (2 * i, 2 * i + 1) if neighbours else (i, i + dims // 2)
            c, s = math.cos(t * fi) * mult, math.sin(t * fi) * mult
            u, v = x[t, :, a], x[t, :, b]
            out[t, :, a] = u * c - v * s
            out[t, :, b] = v * c + u * s
    return out


# ------------------------------------------------------------------------------ convolution
def short_conv(u, w):
    """y_t = sum_j w[:, j] u_{t - taps + 1 + j} per channel; zeros before the start."""
    taps = w.shape[1]
    pad = torch.cat([torch.zeros(taps - 1, u.shape[1], dtype=DT), u], 0)
    return sum(_t(w[:, j]) * pad[j:j + u.shape[0]] for j in range(taps))


def conv_lin(ten, name, h):
    return short_conv(lin(ten, name, h), ten[name + ".conv"])


# ------------------------------------------------------------------------------ mixers
def window_attention(ten, p, m, h):
    """Convolved q, k, v; rotated neighbour pairs; a sliding window; a sink per head in the
    softmax's denominator."""
    T = h.shape[0]
    H, dk = m["heads"], m["dim"]
    G, dv = m.get("kv_heads", H), m.get("vdim", dk)
    q = rotate(conv_lin(ten, p + "q", h).view(T, H, dk), m.get("rot"), True)
    k = rotate(conv_lin(ten, p + "k", h).view(T, G, dk), m.get("rot"), True)
    v = conv_lin(ten, p + "v", h).view(T, G, dv)
    size = (m.get("mask") or {}).get("size", T)
    sink = _t(ten[p + "sink"])
    o = torch.zeros(T, H, dv, dtype=DT)
    for i in range(T):
        first = max(0, i - size + 1)
        for a in range(H):
            g = a // (H // G)
            s = k[first:i + 1, g] @ q[i, a] * m["scale"]
            top = torch.maximum(s.max(), sink[a])
            e = torch.exp(s - top)
            o[i, a] = (e @ v[first:i + 1, g]) / (e.sum() + torch.exp(sink[a] - top))
    return lin(ten, p + "o", o.reshape(T, H * dv))


def retention_core(q, k, v, decay):
    """S_t = decay_h S_{t-1} + k_t v_t^T, o_t = S_t^T q_t; q, k [T, H, dk], v [T, H, dv]."""
    T, H, dk = q.shape
    S = torch.zeros(H, dk, v.shape[-1], dtype=DT)
    d = torch.tensor(decay, dtype=DT)[:, None, None]
    o = torch.zeros(T, H, v.shape[-1], dtype=DT)
    for t in range(T):
        S = d * S + k[t][:, :, None] * v[t][:, None, :]
        o[t] = (S * q[t][:, :, None]).sum(1)
    return o


def retention(ten, p, m, h, eps):
    T = h.shape[0]
    H, dk = m["heads"], m["dim"]
    dv = m.get("vdim", dk)
    q = rotate(lin(ten, p + "q", h).view(T, H, dk), m.get("rot"), False)
    k = rotate(lin(ten, p + "k", h).view(T, H, dk), m.get("rot"), False) * dk ** -0.5
    v = lin(ten, p + "v", h).view(T, H, dv)
    o = rms(retention_core(q, k, v, m["decay"]), eps).reshape(T, H * dv)
    return lin(ten, p + "o", o * silu(lin(ten, p + "g", h)))


def side_by_side(ten, p, m, h, eps):
    return m["left_scale"] * window_attention(ten, p + "left.", m["left"], h) \
        + m["right_scale"] * retention(ten, p + "right.", m["right"], h, eps)


def delta_core(q, k, v, g, beta):
    """S <- g S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q.  q, k [T, G, dk], v
    [T, H, dv], g and beta [T, H]."""
    T, H, dv = v.shape
    rep = H // q.shape[1]
    S = torch.zeros(H, q.shape[2], dv, dtype=DT)
    o = torch.zeros(T, H, dv, dtype=DT)
    for t in range(T):
        for a in range(H):
            kt, qt = k[t, a // rep], q[t, a // rep]
            S[a] = g[t, a] * S[a]
            u = beta[t, a] * (v[t, a] - S[a].T @ kt)
            S[a] = S[a] + kt[:, None] * u[None, :]
            o[t, a] = S[a].T @ qt
    return o


def gated_delta(ten, p, m, h, eps):
    T = h.shape[0]
    H, dk = m["heads"], m["dim"]
    G, dv = m.get("kv_heads", H), m.get("vdim", dk)
    q = silu(conv_lin(ten, p + "q", h)).view(T, G, dk)
    k = silu(conv_lin(ten, p + "k", h)).view(T, G, dk)
    v = silu(conv_lin(ten, p + "v", h)).view(T, H, dv)
    unit = lambda x: x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)   # noqa: E731
    beta = sigmoid(lin(ten, p + "b", h))
    g = torch.exp(-torch.exp(_t(ten[p + "A_log"])) * softplus(lin(ten, p + "a", h) + _t(ten[p + "dt_bias"])))
    o = delta_core(unit(q) * dk ** -0.5, unit(k), v, g, beta)
    o = rms(o, eps) * _t(ten[p + "norm"]) * silu(lin(ten, p + "g", h)).view(T, H, dv)
    return lin(ten, p + "o", o.reshape(T, H * dv))


# ------------------------------------------------------------------------------ feed-forward
def dense(ten, p, h):
    return lin(ten, p + "down", silu(lin(ten, p + "gate", h)) * lin(ten, p + "up", h))


def route(z, top, groups, keep, scale):
    """z [experts] -> [(expert, weight)]."""
    s = sigmoid(z)
    n = s.numel() // groups
    order = sorted(range(groups), key=lambda g: -float(torch.sort(s[g * n:(g + 1) * n], descending=True).values[:2].sum()))
    allowed = [e for g in order[:keep] for e in range(g * n, (g + 1) * n)]
    chosen = sorted(allowed, key=lambda e: -float(s[e]))[:top]
    total = sum(s[e] for e in chosen) + 1e-20
    return [(e, s[e] / total * scale) for e in chosen]


def expert(ten, p, h, limit):
    g = lin(ten, p + "gate", h).clamp(max=limit)
    u = lin(ten, p + "up", h).clamp(-limit, limit)
    return lin(ten, p + "down", g * sigmoid(1.702 * g) * (u + 1.0))


def experts(ten, p, m, h):
    r = m["router"]
    gr = r.get("groups") or {"count": 1, "keep": 1}
    z = lin(ten, p + "router", h)
    y = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, w in route(z[t], r["top"], gr["count"], gr["keep"], r.get("scale", 1.0)):
            y[t] += w * expert(ten, f"{p}e{e}.", h[t:t + 1], m["expert"]["limit"])[0]
    return y


# ------------------------------------------------------------------------------ the model
def forward(cfg, ten, tokens, taps=None):
    """Logits [T, vocab]; ``taps`` (a list) receives the residual after every layer."""
    eps = cfg["norm"]["eps"]
    x = embedding(cfg, ten, list(tokens))
    for i, l in enumerate(cfg["layers"]):
        p, m = f"l{i}.", l["mixer"]
        h = offset_norm(x, ten[p + "norm1"], eps)
        if l["type"] == "parallel":
            x = x + side_by_side(ten, p + "mix.", m, h, eps)
        elif l["type"] == "delta":
            x = x + gated_delta(ten, p + "mix.", m, h, eps)
        else:
            raise ValueError(l["type"])
        if l.get("mlp"):
            h = offset_norm(x, ten[p + "norm2"], eps)
            x = x + (dense(ten, p + "mlp.", h) if l["mlp"]["kind"] == "dense" else experts(ten, p + "mlp.", l["mlp"], h))
        if taps is not None:
            taps.append(x.clone())
    return lin(ten, "head", offset_norm(x, ten["final.norm"], eps))


def layers(cfg, ten, tokens):
    taps = []
    forward(cfg, ten, tokens, taps)
    return taps
