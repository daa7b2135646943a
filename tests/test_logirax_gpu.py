"""Logirax through the engine with the HIP kernels (fp32 sharp, bf16 loose) against the
plain oracle, each mechanism alone, greedy generation through LLMEngine.generate, and the
new kernels against the PyTorch implementation of the same op on multi-segment steps and
inside replayed graphs."""
import os
import sys

import pytest
import torch

sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))
import logirax_cases as C  # noqa: E402
import logirax_engine_cases as E  # noqa: E402
import logirax_mechanism_cases as K  # noqa: E402

pytestmark = pytest.mark.gpu
CASES = [("a", "float32"), ("b", "float32"), ("c", "float32"), ("a", "bfloat16"), ("c", "bfloat16")]


@pytest.mark.parametrize("name,dtype", CASES)
def test_whole_prompt(name, dtype, tmp_path):
    E.whole_prompt(name, "cuda", dtype, tmp_path)


@pytest.mark.parametrize("name", ["a", "b", "c"])
def test_layers(name, tmp_path):
    E.layers_of_a_prompt(name, "cuda", "float32", tmp_path)


@pytest.mark.parametrize("name,dtype", CASES)
def test_prefill_then_decode(name, dtype, tmp_path):
    E.prefill_then_decode(name, "cuda", dtype, tmp_path)


@pytest.mark.parametrize("name", ["a", "c"])
def test_portions(name, tmp_path):
    E.portions_of_a_prompt(name, "cuda", "float32", tmp_path)


@pytest.mark.parametrize("name,dtype", CASES)
def test_mixed_batches_and_reuse(name, dtype, tmp_path):
    E.mixed_batches_and_reuse(name, "cuda", dtype, tmp_path)


def test_peaked_scores(tmp_path):
    E.peaked_scores("cuda", "float32", tmp_path)


def test_shifted_long_decode(tmp_path):
    E.shifted_long_decode("cuda", "float32", tmp_path)


@pytest.mark.parametrize("name", ["a", "b", "c"])
def test_greedy_generation(name, tmp_path):
    E.greedy_generation(name, "cuda", "float32", tmp_path)


@pytest.mark.parametrize("name", ["a", "b", "c"])
def test_greedy_generation_graphs(name, tmp_path):
    """Decode steps replayed from captured graphs and queued ahead of the host."""
    E.greedy_generation(name, "cuda", "float32", tmp_path, graphs=True)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("case", K.CASES)
def test_mechanism(case, dtype):
    K.run(case, "cuda", dtype)


def test_bf16_generation_runs(tmp_path):
    from fasttalk_llm_microservice_amd.engine.sampling_params import SamplingParams

    d, cfg, _ = C.make_model("a", 3, tmp_path)
    eng = C.make_engine(d, "cuda", "bfloat16", seqs=3)
    outs = eng.generate([C.tokens(n, cfg["vocab"], n) for n in (3, 20, 1, 7)],
                        SamplingParams(temperature=0.8, top_p=0.9, max_tokens=9, ignore_eos=True, seed=1))
    assert [len(o) for o in outs] == [9] * 4 and all(0 <= t < cfg["vocab"] for o in outs for t in o)


def _segments(device, rows, pos0, slots, page, pad=0):
    """A step of several sequences (+ ``pad`` empty padding segments with slot -1)."""
    from fasttalk_llm_microservice_amd.ops import mixers as M

    i32 = lambda v: torch.tensor(v, dtype=torch.int32, device=device)   # noqa: E731
    start, tables, slot_map, nb, positions = [0], [], [], 0, []
    maxb = max((p + r + page - 1) // page for p, r in zip(pos0, rows))
    for r, p in zip(rows, pos0):
        n = (p + r + page - 1) // page
        tab = list(range(nb, nb + n)) + [0] * (maxb - n)
        nb += n
        tables.append(tab)
        slot_map += [tab[q // page] * page + q % page for q in range(p, p + r)]
        positions += list(range(p, p + r))
        start.append(start[-1] + r)
    kv = [p + r for p, r in zip(pos0, rows)]
    for _ in range(pad):
        start.append(start[-1])
        tables.append([0] * maxb)
        kv.append(0)
    seg = M.Segments(start=i32(start), pos0=i32(list(pos0) + [0] * pad), slot=i32(list(slots) + [-1] * pad),
                     kv_len=i32(kv), block_tables=i32(tables), num=len(rows) + pad, max_rows=max(rows), max_kv=max(kv))
    return seg, i32(slot_map), i32(positions), nb


def _on(seg, dev):
    from fasttalk_llm_microservice_amd.ops import mixers as M

    return M.Segments(**{**seg.__dict__, **{k: getattr(seg, k).to(dev) for k in
                                            ("start", "pos0", "slot", "kv_len", "block_tables")}})


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H,G,d", [(6, 2, 24), (5, 5, 7), (16, 4, 128), (12, 4, 32), (33, 11, 16), (32, 8, 128), (32, 4, 64),
                                   (24, 3, 40), (20, 20, 72), (16, 1, 160), (8, 1, 264), (64, 4, 32), (64, 8, 128)])
def test_talking_kernels_multi_segment(dtype, H, G, d):
    """The preparation and the per-row attention kernel on a step of unequal segments (decode
    rows deep in a sequence, a fresh prompt, a later portion, padding) against the PyTorch
    implementation, with and without the gate."""
    from fasttalk_llm_microservice_amd.ops import mixers as M

    g = torch.Generator().manual_seed(9)
    page, nq, nk = 8, H * d, G * d
    rows, pos0, slots = [1, 13, 5, 1], [170, 0, 30, 2], [2, 0, 3, 1]
    seg, slot_map, positions, nb = _segments("cuda", rows, pos0, slots, page, pad=2)
    T = sum(rows)
    p = (torch.randn(T, 2 * nq + nk, generator=g) * 0.7).to("cuda", dtype)
    kc0 = (torch.randn(nb, page, nk, generator=g)).to("cuda", dtype)
    vc0 = (torch.randn(nb, page, nk, generator=g) * 0.5).to("cuda", dtype)
    q_scale = (torch.rand(H, generator=g) * 0.3 + 0.1).cuda()
    talk = (torch.eye(H) + 0.3 * torch.randn(H, H, generator=g)).cuda()
    rot = d // 2 // 2 * 2
    table = M.rope_table(256, rot, 1000.0, device="cuda")
    for inter in (False, True):
        outs = []
        for dev in ("cuda", "cpu"):
            mv = lambda t: t.clone().to(dev)   # noqa: E731
            sg = _on(seg, dev)
            kc, vc, pp = mv(kc0), mv(vc0), mv(p)
            spec = M.TalkSpec(H, G, d, d, 150, 5, 6.0, mv(talk))
            q = M.rot_norm_prep(pp, nq, nk, d, mv(table), rot, 1e-5, mv(q_scale), mv(positions), mv(slot_map), kc, vc,
                                interleaved=inter)
            o1 = M.talk_attention(torch.zeros(T, nq, dtype=dtype, device=dev), q, pp[:, nq + nk:], kc, vc, sg, spec)
            o2 = M.talk_attention(torch.zeros(T, nq, dtype=dtype, device=dev), q, None, kc, vc, sg, spec)
            outs.append([t.float().cpu() for t in (q, kc, vc, o1, o2)])
        tol = dict(rtol=3e-5, atol=3e-5) if dtype == torch.float32 else dict(rtol=2e-2, atol=2e-2)
        for a, b, name in zip(outs[0], outs[1], ("q", "k cache", "v cache", "gated attention", "attention")):
            torch.testing.assert_close(a, b, msg=lambda m, n=name: f"{n}: {m}", **tol)


@pytest.mark.parametrize("H,rows,keys,ext", [(1, 5, 40, 0), (6, 33, 100, 7), (16, 12, 257, 3), (20, 9, 64, 0), (40, 4, 90, 11)])
def test_talk_weights_kernel(H, rows, keys, ext):
    from fasttalk_llm_microservice_amd.ops import mixers as M

    g = torch.Generator().manual_seed(2)
    s = torch.randn(H, rows, keys, generator=g) * 4
    talk = torch.eye(H) + 0.3 * torch.randn(H, H, generator=g)
    key0 = ext + 13
    first = key0 + keys - ext - rows
    for window, keep in ((0, 0), (21, ext + 2), (4, ext)):
        if window == 0 and ext:
            continue
        outs = []
        for dev in ("cuda", "cpu"):
            x = s.clone().to(dev)
            inv = M.talk_weights(x, first, key0, ext, M.TalkSpec(H, 1, 8, 8, window, keep, 5.0, talk.to(dev)))
            outs.append((x * inv[:, :, None]).cpu())
        torch.testing.assert_close(outs[0], outs[1], rtol=3e-5, atol=1e-6)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_row_kernels_multi_segment(dtype):
    """The token shift with slot state and the latent preparation on a multi-segment step
    against the PyTorch implementation."""
    from fasttalk_llm_microservice_amd.ops import mixers as M

    g = torch.Generator().manual_seed(10)
    W, page, R, dr, Q, H, dn = 72, 8, 20, 6, 13, 3, 5
    rows, pos0, slots = [1, 13, 5, 1, 2], [17, 0, 30, 0, 1], [2, 0, 3, 1, 4]
    seg, slot_map, positions, nb = _segments("cuda", rows, pos0, slots, page, pad=2)
    T = sum(rows)
    x0, y = torch.randn(T, W, generator=g), torch.randn(T, W, generator=g).to(dtype)
    wb, w, shift = torch.rand(W, generator=g), torch.rand(W, generator=g), torch.rand(W, generator=g)
    st0 = torch.randn(6, W, generator=g)
    p = torch.randn(T, Q + R + dr + 2, generator=g).to(dtype)
    nq_, nkv = 1 + 0.2 * torch.randn(Q, generator=g), 1 + 0.2 * torch.randn(R, generator=g)
    q = torch.randn(T, H * (dn + dr), generator=g).to(dtype)
    table = M.rope_table(64, dr, 100.0)
    outs = []
    for dev in ("cuda", "cpu"):
        mv = lambda t: t.clone().to(dev)   # noqa: E731
        sg = _on(seg, dev)
        st = mv(st0)
        x, h = M.add_norm_shift_rows(mv(x0), mv(y), mv(wb), mv(w), mv(shift), 1e-5, dtype, st, sg)
        cache = torch.zeros(nb, page, R + dr, dtype=dtype, device=dev)
        pp = mv(p)
        cq = M.latent_down_prep(pp[:, :Q], mv(nq_), pp[:, Q:Q + R + dr], mv(nkv), 1e-5, mv(table), dr, mv(positions),
                                mv(slot_map), cache, R, interleaved=True)
        qn, qr = M.latent_q_rope(mv(q), mv(table), dr, mv(positions), H, dn, dr, True)
        outs.append([t.float().cpu() for t in (x, h, st, cq, cache, qn, qr)])
    tol = dict(rtol=3e-5, atol=3e-5) if dtype == torch.float32 else dict(rtol=2e-2, atol=2e-2)
    for a, b, name in zip(outs[0], outs[1], ("residual", "shifted", "state", "query latent", "cache", "qn", "qr")):
        torch.testing.assert_close(a, b, msg=lambda m, n=name: f"{n}: {m}", **tol)
    assert torch.equal(outs[0][2][5], st0[5])                                  # a slot of no sequence


def test_graph_replays_of_new_kernels():
    """Token shift, score-mixing attention and the sigmoid router inside a captured graph:
    several replays with eager work between them give what the eager calls give."""
    from fasttalk_llm_microservice_amd.ops import mixers as M

    g = torch.Generator().manual_seed(4)
    H, G, d, page, W = 4, 2, 16, 8, 48
    nq, nk = H * d, G * d
    seg, slot_map, positions, nb = _segments("cuda", [1, 1, 1], [25, 9, 0], [0, 2, 1], page, pad=1)
    p = torch.randn(3, 2 * nq + nk, generator=g).cuda()
    x0, y = torch.randn(3, W, generator=g).cuda(), torch.randn(3, W, generator=g).cuda()
    wb, w, shift = (torch.rand(W, generator=g).cuda() for _ in range(3))
    router = torch.randn(7, W, generator=g).cuda()
    talk, q_scale = (torch.eye(H) + 0.3 * torch.randn(H, H, generator=g)).cuda(), torch.full((H,), 0.5).cuda()
    spec = M.TalkSpec(H, G, d, d, 6, 2, 5.0, talk)
    kc0, vc0 = torch.randn(nb, page, nk, generator=g).cuda(), torch.randn(nb, page, nk, generator=g).cuda()
    st0 = torch.randn(3, W, generator=g).cuda()
    kc, vc, st, x = kc0.clone(), vc0.clone(), st0.clone(), x0.clone()

    def step():
        xo, h = M.add_norm_shift_rows(x, y, wb, w, shift, 1e-5, torch.float32, st, seg)
        q = M.rot_norm_prep(p, nq, nk, d, None, 0, 1e-5, q_scale, positions, slot_map, kc, vc)
        o = M.talk_attention(torch.empty(3, nq, device="cuda"), q, p[:, nq + nk:], kc, vc, seg, spec)
        idx, wts = M.moe_route_top_logits(h, router, None, 3, True, 1.5)
        return xo, h, o, idx, wts

    def reset():
        kc.copy_(kc0); vc.copy_(vc0); st.copy_(st0); x.copy_(x0)

    want = [t.clone() for t in step()]
    want_st = st.clone()
    torch.cuda.synchronize()
    s = torch.cuda.Stream()
    with torch.cuda.stream(s):
        reset()
        step()
        s.synchronize()
        graph = torch.cuda.CUDAGraph()
        reset()
        with torch.cuda.graph(graph, stream=s):
            out = step()
    for _ in range(3):
        reset()
        graph.replay()
        torch.cuda.synchronize()
        for got, wv in zip(out, want):
            torch.testing.assert_close(got, wv, rtol=1e-6, atol=1e-6)
        torch.testing.assert_close(st, want_st, rtol=1e-6, atol=1e-6)
        _ = (torch.randn(64, 64, device="cuda") @ torch.randn(64, 64, device="cuda")).sum().item()
