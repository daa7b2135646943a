"""Each Logirax mechanism of models/mixers.py (and the ops under it) alone against the
oracle's function for it: one whole sequence, then the same sequence cut in two steps
through the cache / state the first step left; with and without the matrix-product
attention path.  Where random weights would hide a fault, one query and key are scaled so
that a single score stands out just inside or just outside an edge."""
import torch

import logirax_oracle as O

from fasttalk_llm_microservice_amd.models import mixers as X
from fasttalk_llm_microservice_amd.ops import mixers as M

CASES = ["token_shift", "neighbour_rotation", "talking_attention", "talking_attention_products",
         "talking_attention_edges", "talking_attention_far_kept_key", "talking_attention_mix_of_heads",
         "talking_attention_whole_pieces", "latent", "latent_products", "latent_sink", "latent_far_key",
         "latent_head_gate", "router", "experts_pairs", "experts_sorted", "experts_no_shared", "clamped_feed_forward"]
EPS = 1e-5
CFG = {"norm": {"eps": EPS}}


def _rand(g, *shape, s=1.0):
    return (torch.randn(*shape, generator=g) * s).bfloat16().float()


def _ctx(T, device, cut=None, page=4, slot=1, host=False):
    """StepContexts of one sequence of T rows: whole, or [0, cut) then [cut, T)."""
    i32 = lambda v: torch.tensor(v, dtype=torch.int32, device=device)   # noqa: E731
    nb = (T + page - 1) // page
    table = list(range(nb - 1, -1, -1))            # pages in reverse order
    out = []
    for a, b in ([(0, T)] if cut is None else [(0, cut), (cut, T)]):
        pos = list(range(a, b))
        seg = M.Segments(start=i32([0, b - a]), pos0=i32([a]), slot=i32([slot]), kv_len=i32([b]),
                         block_tables=i32([table]), num=1, max_rows=b - a, max_kv=b,
                         host=([0, b - a], [a], [b]) if host else None)
        slots = [table[p // page] * page + p % page for p in pos]
        out.append((a, b, X.StepContext(None, i32(pos), i32(slots), seg)))
    return out


def _close(got, want, dtype):
    """fp32: sharp.  bf16: rounding of the activations, measured against the output's size."""
    want = want.float()
    if dtype == torch.float32:
        torch.testing.assert_close(got, want, rtol=3e-4, atol=3e-4)
    else:
        assert float((got - want).abs().max()) <= 0.05 * float(want.abs().max()) + 0.02


def _run(mix, h, T, device, dtype, cuts, host, want, page=4, rows=None):
    for cut in cuts:
        c = mix.alloc_cache((T + page - 1) // page, page, dtype, 3, device)
        got = torch.cat([mix(h[a:b].to(device, dtype), ctx, c).float().cpu()
                         for a, b, ctx in _ctx(T, device, cut, page=page, host=host)])
        _close(got if rows is None else got[rows], want if rows is None else want[rows], dtype)


def _talk(device, dtype, host, T=45, H=4, G=2, d=10, window=9, keep=3, scale=0.5, cap=6.0, rot=(6, 100.0),
          cuts=(None, 1, 2, 9, 10, 36), tweak=None, rows=None, page=4, W=40):
    g = torch.Generator().manual_seed(3)
    m = {"heads": H, "kv_heads": G, "dim": d, "scale": scale, "softcap": cap,
         "mask": {"size": window, "keep_first": keep}, "rot": {"dims": rot[0], "base": rot[1]}}
    P = {"q": _rand(g, H * d, W, s=0.4), "q.b": _rand(g, H * d, s=0.3), "k": _rand(g, G * d, W, s=0.4),
         "k.b": _rand(g, G * d, s=0.3), "g": _rand(g, H * d, W, s=0.4), "o": _rand(g, W, H * d, s=0.3),
         "o.b": _rand(g, W, s=0.3), "temp": 1 + _rand(g, H, s=0.3), "talk": torch.eye(H) + _rand(g, H, H, s=0.4)}
    P = {k: v.bfloat16().float() for k, v in P.items()}
    h = _rand(g, T, W)
    if tweak:
        tweak(P, h)
    want = O.talking_attention(CFG, P, "", m, h.double())
    mix = X.TalkingHeadsAttention(P.__getitem__, W, H, G, d, window, keep, scale, cap, rot[0], rot[1], EPS, dtype,
                                  device, T + 1)
    _run(mix, h, T, device, dtype, cuts, host, want, page, rows)


def _one_key_stands_out(P, h, at, key):
    """Row ``at``'s query and row ``key``'s key point along one common direction (q and k are
    normed per head): the score of (at, key) dwarfs every other of that row, if the mask
    lets it through; the key's value is large too."""
    W, H = h.shape[1], P["temp"].numel()
    u = torch.zeros(W)
    u[0] = 1.0
    h[:, 0] *= 0.1
    h[at] = 6.0 * u + 0.1 * h[at]
    h[key] = 6.0 * u + 0.1 * h[key]
    P["q"][:, 0] = 2.0
    P["k"][:, 0] = 2.0
    P["temp"].fill_(4.0)
    P["talk"].copy_(torch.eye(H) + 0.0625)


def _latent(device, dtype, host, T=45, H=3, dn=6, dr=4, dv=5, R=12, Q=9, scale=0.4, base=100.0,
            cuts=(None, 1, 2, 13, 36), tweak=None, rows=None, page=4, W=40):
    g = torch.Generator().manual_seed(5)
    m = {"heads": H, "dim": dn, "rot_dim": dr, "vdim": dv, "kv_rank": R, "q_rank": Q, "scale": scale,
         "rot": {"dims": dr, "base": base}}
    P = {"dq": _rand(g, Q, W, s=0.4), "dq.norm": 1 + _rand(g, Q, s=0.2), "uq": _rand(g, H * (dn + dr), Q, s=0.6),
         "dkv": _rand(g, R + dr, W, s=0.4), "dkv.norm": 1 + _rand(g, R, s=0.2), "uk": _rand(g, H * dn, R, s=0.5),
         "uv": _rand(g, H * dv, R, s=0.5), "sink": _rand(g, H), "g": _rand(g, H, W, s=0.4),
         "o": _rand(g, W, H * dv, s=0.4)}
    P = {k: v.bfloat16().float() for k, v in P.items()}
    h = _rand(g, T, W)
    if tweak:
        tweak(P, h)
    want = O.latent_attention(CFG, P, "", m, h.double())
    mix = X.LatentAttention(P.__getitem__, W, H, dn, dr, dv, R, scale, dr, base, EPS, dtype, device, T + 1,
                            q_latent=True, interleaved=True, sink=True, head_gate=True)
    _run(mix, h, T, device, dtype, cuts, host, want, page, rows)


def _experts(device, dtype, T, E=7, top=3, scale=1.7, ff=20, shared=12, W=24):
    g = torch.Generator().manual_seed(6)
    P = {"router": _rand(g, E, W, s=0.5)}
    for at, n in [(f"e{i}.", ff) for i in range(E)] + ([("shared.", shared)] if shared else []):
        P.update({at + "gate": _rand(g, n, W, s=0.3), at + "up": _rand(g, n, W, s=0.3), at + "down": _rand(g, W, n, s=0.3)})
    h = _rand(g, T, W)
    mlp = {"router": {"experts": E, "top": top, "scale": scale}, "expert": {"ff": ff},
           "shared": {"ff": shared} if shared else None}
    want = O.experts(P, "", mlp, h.double())
    ff_ = X.MoEFF(P.__getitem__, E, top, 0.0, 1, 1, None, dtype, device, routing="top_sigmoid", act="silu_glu",
                  shared=bool(shared), shared_gate=False, route_scale=scale)
    _close(ff_(h.to(device, dtype)).float().cpu(), want, dtype)


def run(case, device, dtype):
    g = torch.Generator().manual_seed(1)
    if case == "token_shift":
        # widths that fill one or several register chunks of a row, in whole 16-byte pieces or not
        for width in (24, 50, 2049, 2400, 4100):
            T = 11
            x0, y, wb, w = _rand(g, T, width), _rand(g, T, width), _rand(g, width, s=0.2), _rand(g, width, s=0.2)
            shift = torch.rand(width, generator=g)
            y = y.to(dtype).float()
            x1 = x0.double() + O.offset_norm(y.double(), wb, EPS)
            one = lambda v: (1 + v).to(device)   # noqa: E731
            for use_y in (True, False):
                xw = x1 if use_y else x0.double()
                hw = O.offset_norm(xw, w, EPS)
                want = O.token_shift(hw, shift)
                for cut in (None, 1, 2, 10):
                    state = torch.full((3, width), 7.0, device=device)   # a slot's old row is never read at position 0
                    got, res = [], []
                    for a, b, ctx in _ctx(T, device, cut):
                        x, h = M.add_norm_shift_rows(x0[a:b].clone().to(device), y[a:b].to(device, dtype) if use_y else None,
                                                     one(wb) if use_y else None, one(w), shift.to(device), EPS, dtype,
                                                     state, ctx.seg)
                        got.append(h.float().cpu())
                        res.append(x.cpu())
                    torch.testing.assert_close(torch.cat(res), xw.float(), rtol=2e-5, atol=2e-5)
                    if dtype == torch.float32:
                        torch.testing.assert_close(torch.cat(got), want.float(), rtol=3e-5, atol=3e-5)
                    else:
                        torch.testing.assert_close(torch.cat(got), want.float(), rtol=1e-2, atol=1e-2)
                    torch.testing.assert_close(state[1].cpu(), hw[-1].float(), rtol=2e-5, atol=2e-5)
                    assert float(state[0].min()) == 7.0 and float(state[2].max()) == 7.0   # other slots untouched
    elif case == "neighbour_rotation":
        T, H, dn, dr = 300, 2, 3, 8
        q = _rand(g, T, H * (dn + dr))
        table = M.rope_table(T, dr, 50.0, device=device)
        pos = torch.arange(T, dtype=torch.int32, device=device)
        for inter in (True, False):
            qn, qr = M.latent_q_rope(q.to(device, dtype), table, dr, pos, H, dn, dr, inter)
            v = q.view(T, H, dn + dr).double()
            f = O.rotate_neighbours if inter else O.rotate_half
            torch.testing.assert_close(qn.cpu(), v[..., :dn].float(), rtol=0, atol=0)
            torch.testing.assert_close(qr.cpu(), f(v[..., dn:], {"dims": dr, "base": 50.0}).float(), rtol=1e-4, atol=2e-4)
    elif case == "talking_attention":
        _talk(device, dtype, host=False)
        _talk(device, dtype, host=False, H=3, G=3, d=8, window=1, keep=0, rot=(8, 50.0), cuts=(None, 7))
        _talk(device, dtype, host=False, H=2, G=1, d=80, window=16, keep=40, rot=(0, 1.0), scale=0.1, cuts=(None, 20))
        _talk(device, dtype, host=False, H=1, G=1, d=9, window=100, keep=0, rot=(2, 10.0), cuts=(None, 33))
        _talk(device, dtype, host=False, H=20, G=4, d=8, window=30, keep=1, cuts=(None, 31))   # five heads per key head
        _talk(device, dtype, host=False, H=34, G=17, d=8, window=12, keep=5, cuts=(None, 40))
    elif case == "talking_attention_whole_pieces":
        # head sizes whose rows are whole 16-byte pieces in both dtypes (the kernels' vector loads), and several
        # 64-key tiles per row
        _talk(device, dtype, host=False, T=150, H=8, G=2, d=16, window=100, keep=9, rot=(16, 1000.0), cuts=(None, 120))
        _talk(device, dtype, host=False, T=140, H=6, G=3, d=24, window=130, keep=2, rot=(8, 50.0), cuts=(None, 139))
        _talk(device, dtype, host=False, T=70, H=4, G=4, d=136, window=40, keep=4, rot=(64, 1000.0), scale=0.1,
              cuts=(None, 69))
    elif case == "talking_attention_products":
        _talk(device, dtype, host=True, T=100, cuts=(None, 33, 48, 64))
        _talk(device, dtype, host=True, T=100, window=40, keep=50, cuts=(None, 36, 60))
        _talk(device, dtype, host=True, T=80, window=3, keep=1, cuts=(None, 32))
        _talk(device, dtype, host=True, T=70, H=18, G=6, d=8, window=33, keep=4, cuts=(None, 35))     # two mix tiles
        _talk(device, dtype, host=True, T=64, H=36, G=4, d=8, window=20, keep=0, cuts=(None,))
        _talk(device, dtype, host=True, T=600, H=2, G=1, d=8, window=17, keep=6, cuts=(None, 300))    # several row chunks
    elif case == "talking_attention_edges":
        # window 9, 3 kept: row 40 sees 32..40 and 0..2; the keys at 31 and at 3 must not be seen
        for at, key in ((40, 32), (40, 31), (40, 2), (40, 3), (12, 3), (11, 3), (44, 0)):
            for host in (False, True):
                _talk(device, dtype, host=host, T=46, rot=(0, 1.0),
                      tweak=lambda P, h, at=at, key=key: _one_key_stands_out(P, h, at, key),
                      cuts=(None, 3, 32, 40, 41) if not host else (None, 3), rows=[at])
    elif case == "talking_attention_far_kept_key":
        # hundreds of keys between a kept token and the rows that still see it; page borders in between
        for host in (False, True):
            _talk(device, dtype, host=host, T=400, window=17, keep=2, page=16, rot=(0, 1.0),
                  tweak=lambda P, h: _one_key_stands_out(P, h, 399, 1), cuts=(None, 352, 399), rows=[399, 398, 200])
    elif case == "talking_attention_mix_of_heads":
        # a mix that only moves scores between heads: head 0 attends by head 3's scores and so on; then a mix of
        # large entries of both signs behind a tight cap
        def moved(P, h):
            H = P["temp"].numel()
            P["talk"].zero_()
            for i in range(H):
                P["talk"][i, H - 1 - i] = 4.0

        def signed(P, h):
            P["talk"].copy_(8.0 * torch.sign(P["talk"]))
        for host in (False, True):
            for tw, cap in ((moved, 6.0), (signed, 0.5)):
                _talk(device, dtype if tw is moved else torch.float32, host=host, T=50, window=20, cap=cap, tweak=tw,
                      cuts=(None, 34))
    elif case == "latent":
        _latent(device, dtype, host=False)
        _latent(device, dtype, host=False, H=1, dn=3, dr=2, dv=70, R=70, Q=1, cuts=(None, 7))
        _latent(device, dtype, host=False, H=18, dn=4, dr=8, dv=3, R=8, Q=30, cuts=(None, 20))
    elif case == "latent_products":
        _latent(device, dtype, host=True, T=100, cuts=(None, 33, 64))
        _latent(device, dtype, host=True, T=70, H=5, dn=8, dr=6, dv=8, R=24, Q=16, cuts=(None, 35))
    elif case == "latent_sink":
        # sinks that take nearly all of the weight, none of it, and a share, by head; scores small
        def tweak(P, h):
            P["sink"].copy_(torch.tensor([6.0, -20.0, 1.0]))
            P["uq"].mul_(0.0625)
        for host in (False, True):
            _latent(device, dtype, host=host, T=40, tweak=tweak, cuts=(None, 1, 37))
    elif case == "latent_far_key":
        # one key hundreds of positions back holds the weight of the last rows
        def tweak(P, h):
            u = torch.zeros(h.shape[1])
            u[0] = 1.0
            h[:, 0] *= 0.1
            for r in (399, 398, 5):
                h[r] = 6.0 * u + 0.1 * h[r]
            # one shared direction in both latents: the unrotated parts of rows 5, 398 and 399 align
            P["dq"][:, 0] = 2.0
            P["dkv"][:12, 0] = 2.0
            P["uq"].abs_()
            P["uk"].abs_()
        for host in (False, True):
            _latent(device, dtype, host=host, T=400, tweak=tweak, page=16, cuts=(None, 352, 399), rows=[399, 398, 200])
    elif case == "latent_head_gate":
        o, gate = _rand(g, 3, 17, 10), _rand(g, 17, 8)
        got = M.head_gate(o.to(device), gate.to(device, dtype)[:, 2:5], dtype).float().cpu()
        want = (o.double() * torch.sigmoid(gate.double()[:, 2:5]).t()[:, :, None]).transpose(0, 1).reshape(17, 30)
        _close(got, want, dtype)
    elif case == "router":
        z = _rand(g, 40, 9, s=3.0)
        z[3] = 0.5                                 # ties go to the lower index
        z[4] = -40.0                               # scores that nearly vanish are still renormalised
        z[5, :4] = torch.tensor([30.0, 31.0, 29.0, 28.0])
        for top, scale in ((1, 1.0), (4, 2.5), (9, 0.7)):
            idx, w = M.moe_top_sigmoid(z.to(device), top, scale)
            h, router = _rand(g, 40, 16).to(dtype), _rand(g, 9, 16)
            idx2, w2 = M.moe_route_top_logits(h.to(device), router.to(device), None, top, True, scale)
            for i, wt, zz in ((idx, w, z), (idx2, w2, h.float() @ router.t())):
                for t, chosen in enumerate(O.route(zz.double(), top, scale)):
                    assert i[t].tolist() == [e for e, _ in chosen], (t, i[t].tolist(), chosen)
                    torch.testing.assert_close(wt[t].cpu(), torch.tensor([x for _, x in chosen]), rtol=2e-5, atol=1e-6)
    elif case == "experts_pairs":
        _experts(device, dtype, 5)
        _experts(device, dtype, 64, E=4, top=4, ff=8, shared=40)
        _experts(device, dtype, 3, E=2, top=1, scale=1.0, ff=33, shared=1, W=25)
    elif case == "experts_sorted":
        _experts(device, dtype, 65)
        _experts(device, dtype, 150, E=5, top=1, scale=0.5, ff=16, shared=24)
        _experts(device, dtype, 90, E=3, top=3, ff=9, shared=5, W=25)
    elif case == "experts_no_shared":
        _experts(device, dtype, 9, shared=0)
        _experts(device, dtype, 70, shared=0)
    elif case == "clamped_feed_forward":
        W, ff = 24, 50
        P = {"gate": _rand(g, ff, W, s=0.4), "up": _rand(g, ff, W, s=0.4), "down": _rand(g, W, ff, s=0.4)}
        h = _rand(g, 9, W)
        for limit in (0.3, 1.5, 100.0):            # most, some and none of the entries are clamped
            got = X.GatedFF(P.__getitem__, dtype, device, act="clamp_glu", limit=limit)(h.to(device, dtype)).float().cpu()
            _close(got, O.clamped_glu(P, "", h.double(), limit), dtype)
    else:
        raise ValueError(case)
