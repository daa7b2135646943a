"""Plain, slow implementation of the Logirax design, written from its equations: one
function per mechanism, whole sequences at a time, no cache, no package code.

A model is (cfg, tensors): ``cfg`` the parsed ``config.json`` dict, ``tensors`` a dict of
torch tensors by checkpoint name.  Everything is evaluated in ``DT`` (float64 by default,
so that the comparison's error is the framework's alone).

Notation: T tokens, x the residual [T, width], p = 0..T-1 the positions.
"""
import torch

DT = torch.float64


def _t(x):
    return x.to(DT)


def lin(ten, name, h):
    y = h @ _t(ten[name]).T
    return y + _t(ten[name + ".b"]) if name + ".b" in ten else y


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def offset_norm(x, w, eps):
    """Residual-stream norm: the stored weight is an offset from one."""
    return rms(x, eps) * (1.0 + _t(w))


def token_shift(h, w):
    """h_t moved towards h_{t-1} by w per element; h_{-1} = 0."""
    prev = torch.cat([torch.zeros_like(h[:1]), h[:-1]], 0)
    return h + (prev - h) * _t(w)


# ------------------------------------------------------------------------------ positions
def angles(rot, T):
    half = rot["dims"] // 2
    f = torch.tensor([float(rot["base"]) ** (-2.0 * i / rot["dims"]) for i in range(half)], dtype=DT)
    return torch.arange(T, dtype=DT)[:, None] * f[None]


def rotate_half(x, rot):
    """x [T, heads, dim]: entry i of the first dims entries paired with i + dims/2."""
    dims = (rot or {}).get("dims", 0)
    if not dims:
        return x
    half = dims // 2
    a = angles(rot, x.shape[0])[:, None, :]
    c, s = a.cos(), a.sin()
    out = x.clone()
    u, v = x[..., :half], x[..., half:dims]
    out[..., :half] = u * c - v * s
    out[..., half:dims] = v * c + u * s
    return out


def rotate_neighbours(x, rot):
    """x [T, heads, dim]: entry 2i paired with 2i + 1."""
    dims = (rot or {}).get("dims", 0)
    if not dims:
        return x
    a = angles(rot, x.shape[0])[:, None, :]
    c, s = a.cos(), a.sin()
    out = x.clone()
    u, v = x[..., 0:dims:2], x[..., 1:dims:2]
    out[..., 0:dims:2] = u * c - v * s
    out[..., 1:dims:2] = v * c + u * s
    return out


# ------------------------------------------------------------------------------ masks, softmax
def causal(T):
    return torch.arange(T)[None, :] <= torch.arange(T)[:, None]


def window_visible(mask, T):
    """The last mask.size positions and the first mask.keep_first of the sequence."""
    vis = causal(T)
    if not mask:
        return vis
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    return vis & ((i - j < mask["size"]) | (j < mask.get("keep_first", 0)))


def softmax_sink(s, vis, sink=None):
    """Weights over the visible keys of s [H, T, T]; sink [H]: exp(sink) joins the denominator."""
    s = s.masked_fill(~vis, float("-inf"))
    m = s.max(-1, keepdim=True).values
    if sink is not None:
        m = torch.maximum(m, sink[:, None, None])
    e = torch.exp(s - m)
    d = e.sum(-1, keepdim=True)
    if sink is not None:
        d = d + torch.exp(sink[:, None, None] - m)
    return e / d


# ------------------------------------------------------------------------------ mixers
def talking_scores(s, temp, cap, talk):
    """s [H, T, T] scaled dot products -> per-head factor, tanh cap, mix over the heads."""
    s = s * temp[:, None, None]
    s = cap * torch.tanh(s / cap)
    return torch.einsum("hg,gij->hij", talk, s)


def talking_attention(cfg, ten, p, m, h):
    """Grouped-query attention whose values are its keys as projected; q and k are rotated
    and then normed per head; capped scores are mixed across the heads before the softmax."""
    T = h.shape[0]
    H, G, d = m["heads"], m.get("kv_heads", m["heads"]), m["dim"]
    eps = cfg["norm"]["eps"]
    q = lin(ten, p + "q", h).view(T, H, d)
    k = lin(ten, p + "k", h).view(T, G, d)
    v = k
    q = rms(rotate_half(q, m.get("rot")), eps)
    k = rms(rotate_half(k, m.get("rot")), eps)
    rep = H // G
    s = torch.stack([q[:, a] @ k[:, a // rep].T for a in range(H)]) * m["scale"]
    s = talking_scores(s, _t(ten[p + "temp"]), m["softcap"], _t(ten[p + "talk"]))
    w = softmax_sink(s, window_visible(m.get("mask"), T))
    o = torch.stack([w[a] @ v[:, a // rep] for a in range(H)], 1).reshape(T, H * d)
    return lin(ten, p + "o", o * torch.sigmoid(lin(ten, p + "g", h)))


def latent_attention(cfg, ten, p, m, h):
    """Keys and values are up-projections of one normed latent per token plus one rotated
    key part shared by the heads; queries pass a normed latent of their own; a sink per
    head; a sigmoid gate per head."""
    T = h.shape[0]
    H, dn, dr, dv, R = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    eps = cfg["norm"]["eps"]
    cq = rms(lin(ten, p + "dq", h), eps) * _t(ten[p + "dq.norm"])
    q = lin(ten, p + "uq", cq).view(T, H, dn + dr)
    d = lin(ten, p + "dkv", h)
    c = rms(d[:, :R], eps) * _t(ten[p + "dkv.norm"])
    rot = dict(m["rot"])
    kr = rotate_neighbours(d[:, None, R:], rot)[:, 0]
    qr = rotate_neighbours(q[..., dn:], rot)
    k = lin(ten, p + "uk", c).view(T, H, dn)
    v = lin(ten, p + "uv", c).view(T, H, dv)
    s = torch.stack([q[:, a, :dn] @ k[:, a].T + qr[:, a] @ kr.T for a in range(H)]) * m["scale"]
    w = softmax_sink(s, causal(T), _t(ten[p + "sink"]))
    o = torch.stack([w[a] @ v[:, a] for a in range(H)], 1)
    o = o * torch.sigmoid(lin(ten, p + "g", h))[:, :, None]
    return lin(ten, p + "o", o.reshape(T, H * dv))


# ------------------------------------------------------------------------------ feed-forward
def clamped_glu(ten, p, h, limit):
    g = lin(ten, p + "gate", h).clamp(max=limit)
    u = lin(ten, p + "up", h).clamp(-limit, limit)
    return lin(ten, p + "down", g * torch.sigmoid(1.702 * g) * (u + 1))


def silu_expert(ten, p, h):
    g = lin(ten, p + "gate", h)
    return lin(ten, p + "down", g * torch.sigmoid(g) * lin(ten, p + "up", h))


def route(z, top, scale):
    """Per token: the chosen experts and their weights (sigmoid scores, renormalised, scaled)."""
    s = torch.sigmoid(z)
    out = []
    for t in range(z.shape[0]):
        order = sorted(range(z.shape[1]), key=lambda e: (-float(z[t, e]), e))[:top]
        tot = sum(float(s[t, e]) for e in order) + 1e-20
        out.append([(e, float(s[t, e]) / tot * scale) for e in order])
    return out


def experts(ten, p, mlp, h):
    r = mlp["router"]
    out = torch.zeros_like(h)
    for t, chosen in enumerate(route(lin(ten, p + "router", h), r["top"], r["scale"])):
        for e, w in chosen:
            out[t] += w * silu_expert(ten, f"{p}e{e}.", h[t:t + 1])[0]
    if mlp.get("shared"):
        out = out + silu_expert(ten, p + "shared.", h)
    return out


# ------------------------------------------------------------------------------ the model
def forward(cfg, ten, tokens, taps=None):
    """Logits [T, vocab]; ``taps`` (a list) receives the residual after every layer."""
    eps = cfg["norm"]["eps"]
    x = _t(ten["embed"])[list(tokens)] * cfg["embedding"]["scale"]
    for i, l in enumerate(cfg["layers"]):
        p = f"l{i}."
        h = token_shift(offset_norm(x, ten[p + "norm1"], eps), ten[p + "shift"])
        mix = {"attention": talking_attention, "latent_attention": latent_attention}[l["type"]]
        x = x + offset_norm(mix(cfg, ten, p + "mix.", l["mixer"], h), ten[p + "norm1b"], eps)
        f = l.get("mlp")
        if f:
            h = offset_norm(x, ten[p + "norm2"], eps)
            y = clamped_glu(ten, p + "mlp.", h, f["limit"]) if f["kind"] == "dense" else \
                experts(ten, p + "mlp.", f, h)
            x = x + offset_norm(y, ten[p + "norm2b"], eps)
        if taps is not None:
            taps.append(x.clone())
    h = offset_norm(x, ten["final.norm"], eps)
    return h @ _t(ten["embed"]).T * cfg.get("logit_scale", 1.0)


def greedy(cfg, ten, prompt, n):
    toks = list(prompt)
    for _ in range(n):
        toks.append(int(forward(cfg, ten, toks)[-1].argmax()))
    return toks[len(prompt):]


def layers(cfg, ten, tokens):
    taps = []
    forward(cfg, ten, tokens, taps)
    return taps
