"""Each Pitelorn mechanism of models/mixers.py (and the ops under it) alone against the
oracle's function for it: one whole sequence, then the same sequence cut in two steps
through the cache / state the first step left; with and without the matrix-product
attention path.  Where random weights would hide a fault, one query and key are scaled so
that a single score stands out just inside or just outside an edge, keys are made nearly
equal, or decays set so that what a far token wrote still dominates."""
import torch

import pitelorn_oracle as O
from fufipel_mechanism_cases import _close, _ctx, _one_key_stands_out, _rand, _run

from fasttalk_llm_microservice_amd.models import mixers as X
from fasttalk_llm_microservice_amd.ops import mixers as M

CASES = ["pair_embedding", "plain_residual_add", "window_attention", "window_attention_products",
         "window_attention_edges", "window_attention_sinks", "rotation_pairs", "retention", "retention_odd_sizes",
         "retention_chunk_edges", "retention_far_token", "side_by_side_scales", "delta", "delta_odd_sizes",
         "delta_chunk_edges", "delta_equal_keys", "delta_decays", "delta_far_token", "routing", "routing_many_rows",
         "experts", "dense_feed_forward"]
EPS = 1e-5
W = 40


def _attention_weights(g, H, G, dk, dv, taps):
    P = {"q": _rand(g, H * dk, W, s=0.4), "k": _rand(g, G * dk, W, s=0.4), "v": _rand(g, G * dv, W, s=0.4),
         "o": _rand(g, W, H * dv, s=0.3), "sink": _rand(g, H)}
    for n, c in (("q", H * dk), ("k", G * dk), ("v", G * dv)):
        P[n + ".conv"] = _rand(g, c, taps, s=0.5)
    return P


def _attention_mixer(P, m, device, dtype, max_pos):
    rot = m.get("rot") or {}
    sc = rot.get("scaling")
    return X.ConvSinkAttention(
        P.__getitem__, W, m["heads"], m["kv_heads"], m["dim"], m["vdim"], P["q.conv"].shape[1], m["scale"], 0.0, EPS,
        dtype, device, window=m["mask"]["size"], sink="learned", qk_norm=False, rot_dims=rot.get("dims", 0),
        rot_base=rot.get("base", 1e4), rot_ramp=tuple(sc[k] for k in ("factor", "original", "fast", "slow")) if sc else None,
        interleaved=True, max_pos=max_pos)


def _attention(device, dtype, host, T=45, H=4, G=2, dk=12, dv=7, window=9, taps=3, scale=0.3, rot=None,
               cuts=(None, 1, 2, 9, 10, 36), tweak=None, rows=None, page=4):
    g = torch.Generator().manual_seed(3)
    rot = rot if rot is not None else {"dims": 8, "base": 100.0,
                                       "scaling": {"factor": 4.0, "original": 32, "fast": 4.0, "slow": 0.5}}
    m = {"heads": H, "kv_heads": G, "dim": dk, "vdim": dv, "scale": scale, "mask": {"size": window}, "rot": rot}
    P = _attention_weights(g, H, G, dk, dv, taps)
    h = _rand(g, T, W)
    if tweak:
        tweak(P, h)
    want = O.window_attention(P, "", m, h.double())
    mix = _attention_mixer(P, m, device, dtype, T + 1)
    for cut in cuts:
        cache = mix.alloc_cache((T + page - 1) // page, page, dtype, 3, device)
        cache[2].fill_(7.0)                          # a slot's old history is never read at position 0
        _run(mix, h, T, device, dtype, (cut,), host, page, cache=cache, rows=rows, want=want)
        if taps > 1:
            assert float(cache[2][0].min()) == 7.0 and float(cache[2][2].max()) == 7.0    # other slots untouched


def _identity_convolutions(P):
    for n in ("q.conv", "k.conv", "v.conv"):
        P[n].zero_()
        P[n][:, -1] = 1.0


def _retention_model(g, H, dk, dv):
    return {"q": _rand(g, H * dk, W, s=0.4), "k": _rand(g, H * dk, W, s=0.4), "v": _rand(g, H * dv, W, s=0.4),
            "g": _rand(g, H * dv, W, s=0.4), "o": _rand(g, W, H * dv, s=0.3)}


def _state_mixer(mix, h, T, device, dtype, cuts, want, of=lambda c: c, fill=True, host=True):
    for cut in cuts:
        state = mix.alloc_cache(1, 4, dtype, 3, device)
        parts = [t for t in ([state] if isinstance(state, torch.Tensor) else state) if t.numel()]
        for t in parts:
            t.fill_(7.0)                             # a slot's old state is never read at position 0
        got = torch.cat([mix(h[a:b].to(device, dtype), ctx, state).float().cpu()
                         for a, b, ctx in _ctx(T, device, cut, host=host)])
        _close(got, want, dtype)
        for t in parts:
            assert float(t[0].min()) == 7.0 and float(t[2].max()) == 7.0    # other slots untouched


def _retention(device, dtype, T=45, H=3, dk=10, dv=20, decay=(0.9, 0.97, 0.999), rot=(6, 100.0), cuts=(None, 1, 2, 13, 36),
               tweak=None):
    g = torch.Generator().manual_seed(5)
    m = {"heads": H, "dim": dk, "vdim": dv, "decay": list(decay)[:H], "rot": {"dims": rot[0], "base": rot[1]}}
    P = _retention_model(g, H, dk, dv)
    h = _rand(g, T, W)
    if tweak:
        tweak(P, h)
    want = O.retention(P, "", m, h.double(), EPS)
    mix = X.Retention(P.__getitem__, W, H, dk, dv, m["decay"], rot[0], rot[1], EPS, dtype, device, T + 1)
    _state_mixer(mix, h, T, device, dtype, cuts, want)


def _delta(device, dtype, T=45, H=4, G=2, dk=12, dv=20, taps=3, cuts=(None, 1, 2, 13, 36), tweak=None):
    g = torch.Generator().manual_seed(6)
    m = {"heads": H, "kv_heads": G, "dim": dk, "vdim": dv}
    P = {"q": _rand(g, G * dk, W, s=0.4), "k": _rand(g, G * dk, W, s=0.4), "v": _rand(g, H * dv, W, s=0.4),
         "g": _rand(g, H * dv, W, s=0.4), "a": _rand(g, H, W, s=0.3), "b": _rand(g, H, W, s=0.4), "A_log": _rand(g, H) - 2.0,
         "dt_bias": _rand(g, H), "norm": 1 + _rand(g, dv, s=0.2), "o": _rand(g, W, H * dv, s=0.3)}
    for n, c in (("q", G * dk), ("k", G * dk), ("v", H * dv)):
        P[n + ".conv"] = _rand(g, c, taps, s=0.5)
    h = _rand(g, T, W)
    if tweak:
        tweak(P, h)
    want = O.gated_delta(P, "", m, h.double(), EPS)
    mix = X.HeadDelta(P.__getitem__, W, H, G, dk, dv, taps, EPS, dtype, device)
    _state_mixer(mix, h, T, device, dtype, cuts, want)


def run(case, device, dtype):
    g = torch.Generator().manual_seed(1)
    i32 = lambda v: torch.tensor(v, dtype=torch.int32, device=device)   # noqa: E731
    if case == "pair_embedding":
        # multipliers whose products pass 32 bits; the previous token comes from the slot
        for width, buckets, mp, mc in ((20, 13, 5, 3), (70, 1, 1, 1), (33, 11, 2000003, 1700001)):
            table, pair = _rand(g, 5000, width), _rand(g, buckets + 1, width)
            toks = [3, 0, 4999, 3, 7, 7, 4998, 48]
            cfg = {"embedding": {"bigram": {"buckets": buckets, "mul_prev": mp, "mul_cur": mc}}}
            want = O.embedding(cfg, {"embed": table, "bigram": pair}, toks).float()
            for cut in (None, 1, 5):
                last = i32([44, 45, 46])
                got = [M.pair_embed_rows(ctx.ids, table.to(device, dtype), 1.0, pair.to(device, dtype), mp, mc, buckets,
                                         ctx.seg, last).cpu() for a, b, ctx in _ctx(len(toks), device, cut, ids=toks)]
                torch.testing.assert_close(torch.cat(got), want, rtol=1e-5, atol=1e-5)
                assert last.tolist() == [44, toks[-1], 46]
    elif case == "plain_residual_add":
        for width in (24, 200, 777):
            x0, y, w = _rand(g, 5, width), _rand(g, 5, width), _rand(g, width, s=0.2)
            x = x0.clone().to(device)
            h, _ = M.add_rms_norm_rows(x, y.to(device, dtype), None, EPS, next_w=(1 + w).to(device), out_dtype=dtype)
            torch.testing.assert_close(x.cpu(), x0 + y, rtol=1e-6, atol=1e-6)
            _close(h.float().cpu(), O.offset_norm((x0 + y).double(), w, EPS), dtype)
            assert M.add_rms_norm_rows(x, y.to(device, dtype), None, EPS, out_dtype=dtype) == (None, None)
            torch.testing.assert_close(x.cpu(), x0 + 2 * y, rtol=1e-6, atol=1e-6)
    elif case == "window_attention":
        _attention(device, dtype, host=False)
        _attention(device, dtype, host=False, H=3, G=3, dk=8, dv=72, window=1, taps=1, rot={}, cuts=(None, 7))
        _attention(device, dtype, host=False, H=2, G=1, dk=80, dv=8, window=16, taps=5, scale=0.1,
                   rot={"dims": 80, "base": 50.0}, cuts=(None, 3, 20))
        _attention(device, dtype, host=False, window=100, taps=2)
    elif case == "window_attention_products":
        _attention(device, dtype, host=True, T=100, cuts=(None, 33, 48, 64))
        _attention(device, dtype, host=True, T=100, window=40, taps=4, cuts=(None, 36, 60))
        _attention(device, dtype, host=True, T=80, window=3, cuts=(None, 32))
    elif case == "window_attention_edges":
        # window 9: row 40 sees 32 .. 40; the key at 31 must not be seen however large its score
        for at, key in ((40, 32), (40, 31), (8, 0), (9, 0), (44, 36), (16, 7), (16, 8)):
            for host in (False, True):
                def tweak(P, h, at=at, key=key):
                    _identity_convolutions(P)
                    _one_key_stands_out(P, h, at, key)
                _attention(device, dtype, host=host, T=46, tweak=tweak, rot={},
                           cuts=(None, 3, 32, 40, 41) if not host else (None, 3), rows=[at])
    elif case == "window_attention_sinks":
        for host in (False, True):
            for s in (4.0, -20.0):
                def tweak(P, h, s=s):
                    P["sink"] = torch.tensor([s, 0.0, -s, 1.5])
                _attention(device, dtype, host=host, T=70, window=33, tweak=tweak, cuts=(None, 34))
    elif case == "rotation_pairs":
        # neighbour pairs (interleaved) with the ramp against half pairs without it
        for rot, inter in (({"dims": 8, "base": 100.0, "scaling": {"factor": 4.0, "original": 32, "fast": 4.0, "slow": 0.5}},
                            True), ({"dims": 6, "base": 1000.0}, True), ({"dims": 6, "base": 1000.0}, False)):
            T, H, dk = 20, 2, 10
            x = _rand(g, T, 3 * H * dk)
            sc = rot.get("scaling")
            table = M.rope_table(T, rot["dims"], rot["base"], device=device,
                                 ramp=tuple(sc[k] for k in ("factor", "original", "fast", "slow")) if sc else None)
            (a, b, ctx), = _ctx(T, device)
            kc, vc = (torch.zeros(5, 4, H * dk, dtype=dtype, device=device) for _ in range(2))
            hist = torch.zeros(3, 0, 3 * H * dk, device=device)
            q = M.conv_attn_prep(x.to(device, dtype), H * dk, H * dk, torch.ones(3 * H * dk, 1, device=device), hist,
                                 ctx.seg, None, None, EPS, dk, ctx.slot_mapping, kc, vc, table, rot["dims"], inter)
            want = O.rotate(x[:, :H * dk].double().view(T, H, dk), rot, inter).reshape(T, -1)
            torch.testing.assert_close(q.cpu(), want.float(), rtol=1e-4, atol=1e-4)
            rows = kc.view(-1, H * dk)[ctx.slot_mapping.long()].float().cpu()
            _close(rows, O.rotate(x[:, H * dk:2 * H * dk].double().view(T, H, dk), rot, inter).reshape(T, -1), dtype)
    elif case == "retention":
        _retention(device, dtype)
        _retention(device, dtype, T=100, cuts=(None, 31, 32, 50, 99))
    elif case == "retention_odd_sizes":
        _retention(device, dtype, T=70, H=1, dk=3, dv=33, rot=(2, 10.0), cuts=(None, 20))
        _retention(device, dtype, T=70, H=2, dk=20, dv=65, rot=(0, 10.0), cuts=(None, 17, 36))
        _retention(device, dtype, T=70, H=2, dk=72, dv=8, rot=(72, 1000.0), cuts=(None, 34))
        _retention(device, dtype, T=70, H=1, dk=128, dv=132, rot=(64, 1000.0), cuts=(None, 33))
        _retention(device, dtype, T=70, H=1, dk=200, dv=12, rot=(100, 1000.0), cuts=(None, 33))   # walked at any length
    elif case == "retention_chunk_edges":
        for T in (32, 63, 64, 65, 128, 129, 150):
            _retention(device, dtype, T=T, cuts=(None,) if T < 100 else (None, 64, 65, T - 1))
    elif case == "retention_far_token":
        # a loud first token and slow decays: it dominates every later row, across chunks and cuts
        def loud(P, h):
            h[0] *= 8.0
        _retention(device, dtype, T=150, decay=(0.9999, 1.0, 0.999), cuts=(None, 1, 2, 64, 149), tweak=loud)
    elif case == "side_by_side_scales":
        a = {"heads": 4, "kv_heads": 2, "dim": 12, "vdim": 10, "scale": 0.3, "mask": {"size": 9},
             "rot": {"dims": 8, "base": 100.0}}
        b = {"heads": 3, "dim": 10, "vdim": 14, "decay": [0.9, 0.97, 0.999], "rot": {"dims": 6, "base": 100.0}}
        PL, PR = _attention_weights(g, 4, 2, 12, 10, 3), _retention_model(g, 3, 10, 14)
        both = {**{"left." + k: v for k, v in PL.items()}, **{"right." + k: v for k, v in PR.items()}}
        for ls, rs in ((1.2, 0.5), (1.0, 1.0), (-0.7, 0.0), (0.0, 2.0)):
            T = 70
            h = _rand(g, T, W)
            want = O.side_by_side(both, "", {"left": a, "right": b, "left_scale": ls, "right_scale": rs}, h.double(), EPS)
            for cut in (None, 1, 33, 40):
                mix = X.SideBySideSum(_attention_mixer(PL, a, device, dtype, T + 1),
                                      X.Retention(PR.__getitem__, W, 3, 10, 14, b["decay"], 6, 100.0, EPS, dtype, device,
                                                  T + 1), ls, rs, dtype, device)
                _run(mix, h, T, device, dtype, (cut,), True, want=want)
    elif case == "delta":
        _delta(device, dtype)
        _delta(device, dtype, T=100, cuts=(None, 31, 32, 50, 99))
    elif case == "delta_odd_sizes":
        _delta(device, dtype, T=70, H=1, G=1, dk=3, dv=33, taps=1, cuts=(None, 20))
        _delta(device, dtype, T=70, H=6, G=2, dk=20, dv=65, taps=2, cuts=(None, 17, 36))
        _delta(device, dtype, T=70, H=2, G=2, dk=72, dv=8, taps=5, cuts=(None, 3, 34))
        _delta(device, dtype, T=70, H=2, G=1, dk=128, dv=132, taps=4, cuts=(None, 33))
        _delta(device, dtype, T=70, H=2, G=1, dk=200, dv=12, taps=4, cuts=(None, 33))              # walked at any length
    elif case == "delta_chunk_edges":
        for T in (32, 63, 64, 65, 128, 129, 150):
            _delta(device, dtype, T=T, cuts=(None,) if T < 100 else (None, 64, 65, T - 1))
    elif case == "delta_equal_keys":
        # nearly equal keys and steps near 1: every row overwrites the one before
        def tweak(P, h):
            h[:, 0] = 5.0
            P["k"] *= 0.05
            P["k"][:, 0] = 1.0
            P["b"][:, 0] = 1.5
        _delta(device, dtype, T=140, tweak=tweak, cuts=(None, 70))
    elif case == "delta_decays":
        # heads that forget at once beside heads that hardly forget
        def tweak(P, h):
            P["A_log"] = torch.tensor([-9.0, 3.0, 5.0, -2.0])
            P["dt_bias"] = torch.tensor([0.0, 2.0, 6.0, -8.0])
        _delta(device, dtype, T=140, tweak=tweak, cuts=(None, 1, 70, 139))
    elif case == "delta_far_token":
        # decays and steps near 0: what a loud early token wrote is read by every later row
        def tweak(P, h):
            P["A_log"].fill_(-12.0)
            P["b"][:, 0] = -3.0
            h[:, 0] = 1.0
            h[2, 0] = -6.0
            h[2, 1:] *= 4.0
        _delta(device, dtype, T=150, tweak=tweak, cuts=(None, 3, 64, 149))
    elif case in ("routing", "routing_many_rows"):
        n = 9 if case == "routing" else 130
        for E, top, groups, keep, scale in ((12, 2, 3, 2, 2.5), (6, 6, 1, 1, 1.0), (8, 3, 8, 4, 0.7), (10, 1, 5, 1, 1.3),
                                            (64, 6, 8, 3, 1.0), (130, 4, 13, 5, 2.0), (9, 4, 3, 3, 1.0)):
            P = {"router": _rand(g, E, W, s=0.5)}
            h = _rand(g, n, W)
            z = h.double() @ P["router"].double().T
            hd = h.to(device, dtype)
            if case == "routing":
                idx, wts = M.moe_route_top_logits(hd, P["router"].to(device), None, top, True, scale, groups, keep)
            else:
                idx, wts = M.moe_top_sigmoid(z.float().to(device), top, scale, groups, keep)
            for t in range(n):
                want = O.route(z[t], top, groups, keep, scale)
                assert idx[t].tolist() == [e for e, _ in want]
                torch.testing.assert_close(wts[t].cpu(), torch.stack([w for _, w in want]).float(), rtol=1e-4, atol=1e-5)
    elif case == "experts":
        # few rows (per-pair kernels) and many (grouped products); a limit that clips both ways
        for ff, limit in ((24, 0.3), (16, 100.0)):
            P = {"router": _rand(g, 6, W, s=0.5)}
            for e in range(6):
                P.update({f"e{e}.gate": _rand(g, ff, W, s=0.4), f"e{e}.up": _rand(g, ff, W, s=0.4),
                          f"e{e}.down": _rand(g, W, ff, s=0.4)})
            m = {"router": {"experts": 6, "top": 2, "scale": 1.6, "groups": {"count": 3, "keep": 2}}, "expert": {"limit": limit}}
            mix = X.MoEFF(P.__getitem__, 6, 2, limit, 3, 2, None, dtype, device, routing="top_sigmoid", act="clamp_glu",
                          route_scale=1.6)
            for n in (7, 100):
                h = _rand(g, n, W)
                _close(mix(h.to(device, dtype)).float().cpu(), O.experts(P, "", m, h.double()), dtype)
    elif case == "dense_feed_forward":
        P = {"gate": _rand(g, 50, W, s=0.4), "up": _rand(g, 50, W, s=0.4), "down": _rand(g, W, 50, s=0.4)}
        h = _rand(g, 9, W)
        got = X.GatedFF(P.__getitem__, dtype, device, act="silu")(h.to(device, dtype)).float().cpu()
        _close(got, O.dense(P, "", h.double()), dtype)
    else:
        raise ValueError(case)
