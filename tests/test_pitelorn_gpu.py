"""Pitelorn through the engine with the HIP kernels (fp32 sharp, bf16 loose) against the
plain oracle, each mechanism alone, greedy generation through LLMEngine.generate, and the
new kernels against the PyTorch implementation of the same op on multi-segment steps and
inside replayed graphs."""
import os
import sys

import pytest
import torch

sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))
import pitelorn_cases as C  # noqa: E402
import pitelorn_engine_cases as E  # noqa: E402
import pitelorn_mechanism_cases as K  # noqa: E402
from test_logirax_gpu import _on, _segments  # noqa: E402

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


@pytest.mark.parametrize("name", ["a", "b", "c"])
def test_portions(name, tmp_path):
    E.portions_of_a_prompt(name, "cuda", "float32", tmp_path)


@pytest.mark.parametrize("name,dtype", CASES)
def test_mixed_batches_and_reuse(name, dtype, tmp_path):
    E.mixed_batches_and_reuse(name, "cuda", dtype, tmp_path)


def test_peaked_scores(tmp_path):
    E.peaked_scores("cuda", "float32", tmp_path)


def test_raised_and_lowered_sinks(tmp_path):
    E.raised_and_lowered_sinks("cuda", "float32", tmp_path)


def test_slow_decay_long_decode(tmp_path):
    E.slow_decay_long_decode("cuda", "float32", tmp_path)


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


def _compare(fn, dtype, names, tol32=3e-5):
    """fn(device) -> tensors; the kernels' against the PyTorch implementation's."""
    got, want = ([t.float().cpu() for t in fn(dev)] for dev in ("cuda", "cpu"))
    for a, b, name in zip(got, want, names):
        if dtype == torch.float32:
            torch.testing.assert_close(a, b, rtol=tol32, atol=tol32, msg=lambda m, n=name: f"{n}: {m}")
        else:
            torch.testing.assert_close(a, b, rtol=2e-2, atol=2e-2, msg=lambda m, n=name: f"{n}: {m}")


@pytest.mark.parametrize("H,G,dk,dv", [(4, 2, 16, 16), (6, 2, 20, 33), (3, 3, 64, 72), (4, 1, 128, 128), (2, 2, 100, 8),
                                       (2, 1, 160, 40)])
def test_delta_kernels_multi_segment(H, G, dk, dv):
    """Decode rows deep in a sequence, short and long fresh prompts, later portions on both sides
    of the chunk form's first length, padding segments: conv_delta_prep and head_delta_rule."""
    from fasttalk_llm_microservice_amd.ops import mixers as M

    g = torch.Generator().manual_seed(9)
    taps = 4
    rows, pos0, slots = [1, 13, 70, 1, 150, 33, 31], [170, 0, 30, 2, 0, 5, 64], [2, 0, 3, 1, 5, 4, 6]
    seg, _, _, _ = _segments("cuda", rows, pos0, slots, 8, pad=2)
    T = sum(rows)
    n, nv = G * dk, H * dv
    for dtype in (torch.float32, torch.bfloat16):
        p = (torch.randn(T, 2 * n + nv + 2 * H + 8, generator=g)).to(dtype)
        conv_w = torch.randn(2 * n + nv, taps, generator=g) * 0.5
        hist0, state0 = torch.randn(7, taps - 1, 2 * n + nv, generator=g), torch.randn(7, H, dk, dv, generator=g) * 0.3
        a_log, dt = torch.randn(H, generator=g) - 2, torch.randn(H, generator=g)

        def prep(dev):
            pp, hist = p.to(dev), hist0.clone().to(dev)
            c = 2 * n + nv
            out = M.conv_delta_prep(pp[:, :c], pp[:, c:c + H], pp[:, c + H:c + 2 * H], conv_w.to(dev), hist, a_log.to(dev),
                                    dt.to(dev), _on(seg, dev), H, G, dk, dv)
            return list(out) + [hist]

        _compare(prep, torch.float32, ("q", "k", "v", "log decay", "beta", "history"))
    q, k, v, lg, beta, _ = [t.cpu() for t in prep("cpu")]

    def rule(dev):
        state = state0.clone().to(dev)
        o = M.head_delta_rule(q.to(dev), k.to(dev), v.to(dev), lg.to(dev), beta.to(dev), state, _on(seg, dev))
        return o, state

    _compare(rule, torch.float32, ("o", "state"), tol32=1e-4)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H,dk,dv,rot,inter", [(4, 16, 16, 16, False), (3, 20, 33, 8, True), (2, 64, 72, 0, False),
                                               (3, 128, 128, 128, False), (2, 100, 8, 40, True), (1, 160, 40, 160, False)])
def test_retention_kernels_multi_segment(dtype, H, dk, dv, rot, inter):
    from fasttalk_llm_microservice_amd.ops import mixers as M

    g = torch.Generator().manual_seed(10)
    rows, pos0, slots = [1, 13, 70, 1, 150, 33, 31], [170, 0, 30, 2, 0, 5, 64], [2, 0, 3, 1, 5, 4, 6]
    seg, _, _, _ = _segments("cuda", rows, pos0, slots, 8, pad=2)
    T = sum(rows)
    p = (torch.randn(T, H * (2 * dk + 2 * dv), generator=g) * 0.7).to(dtype)
    state0 = torch.randn(7, H, dk, dv, generator=g)
    ld = torch.log(torch.tensor([0.9995, 0.97, 0.6, 1.0][:H], dtype=torch.float64))
    table = M.rope_table(256, rot, 1000.0) if rot else None
    scale = 0.1 if dk > 64 else 0.3                # outputs of order one

    def run(dev):
        state = state0.clone().to(dev)
        o = M.retention((p * scale).to(dev), table.to(dev) if rot else None, rot, ld.to(dev), state, _on(seg, dev), H, dk, dv,
                        interleaved=inter)
        return o, state

    _compare(run, torch.float32, ("o", "state"), tol32=1e-4)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_attention_kernels_multi_segment(dtype):
    """Convolution, rotation and cache write, and the per-row attention and the banded weights with
    a sink per head."""
    from fasttalk_llm_microservice_amd.ops import mixers as M

    g = torch.Generator().manual_seed(11)
    H, G, dk, dv, page, taps = 6, 2, 24, 40, 8, 4
    nq, nk, nv = H * dk, G * dk, G * dv
    rows, pos0, slots = [1, 13, 5, 1], [70, 0, 30, 2], [2, 0, 3, 1]
    seg, slot_map, _, nb = _segments("cuda", rows, pos0, slots, page, pad=2)
    T = sum(rows)
    p = (torch.randn(T, nq + nk + nv, generator=g) * 0.7).to(dtype)
    conv_w, hist0 = torch.randn(nq + nk + nv, taps, generator=g) * 0.5, torch.randn(4, taps - 1, nq + nk + nv, generator=g)
    kc0 = (torch.randn(nb, page, nk, generator=g) * 0.5).to(dtype)
    vc0 = (torch.randn(nb, page, nv, generator=g) * 0.5).to(dtype)
    table = M.rope_table(128, 16, 1000.0, ramp=(4.0, 64, 4.0, 1.0))
    sinks = torch.randn(H, generator=g) * 3
    wq = torch.rand(dk, generator=g)
    s0 = torch.randn(G, H // G * 5, 40, generator=g)
    for norm in (False, True):
        def run(dev):
            mv = lambda t: t.clone().to(dev)   # noqa: E731
            sg, kc, vc, hist = _on(seg, dev), mv(kc0), mv(vc0), mv(hist0)
            q = M.conv_attn_prep(mv(p), nq, nk, mv(conv_w), hist, sg, mv(wq) if norm else None, mv(wq) if norm else None,
                                 1e-5, dk, mv(slot_map), kc, vc, mv(table), 16, True)
            spec = M.WindowSpec(H, G, dk, dv, 11, 0.2, sink=mv(sinks))
            o = M.window_attention(q, kc, vc, sg, spec)
            return q, kc, vc, hist, o, M.band_weights(mv(s0), 37, 5, spec, 5)

        _compare(run, dtype, ("q", "k cache", "v cache", "history", "attention", "weights"))


@pytest.mark.parametrize("H,G,dk,dv,window", [(16, 4, 128, 128, 150), (6, 2, 24, 40, 100), (32, 8, 64, 64, 0), (5, 5, 16, 8, 1),
                                              (24, 3, 40, 72, 64), (64, 8, 32, 32, 65), (2, 1, 256, 256, 0)])
@pytest.mark.parametrize("sink", ["none", "one", "heads"])
def test_plain_attention_on_key_tiles(H, G, dk, dv, window, sink):
    """bf16 decode rows and short segments on the head-mixing attention's key tiles, without a mix:
    window or every earlier key, cap, sinks, padding segments."""
    from fasttalk_llm_microservice_amd.ops import mixers as M

    g = torch.Generator().manual_seed(13)
    page = 8
    rows, pos0, slots = [1, 13, 5, 1], [270, 0, 30, 2], [2, 0, 3, 1]
    seg, _, _, nb = _segments("cuda", rows, pos0, slots, page, pad=2)
    T = sum(rows)
    q = torch.randn(T, H * dk, generator=g)
    kc = torch.randn(nb, page, G * dk, generator=g).bfloat16()
    vc = (torch.randn(nb, page, G * dv, generator=g) * 0.5).bfloat16()
    sinks = torch.randn(H, generator=g) * 3
    for cap in (0.0, 4.0):
        def run(dev):
            s = {"none": None, "one": 1.5, "heads": sinks.to(dev)}[sink]
            spec = M.WindowSpec(H, G, dk, dv, window, 1.5 * dk ** -0.5, softcap=cap, sink=s)
            assert M._plain_tiles(spec, kc)
            return (M.window_attention(q.to(dev), kc.to(dev), vc.to(dev), _on(seg, dev), spec),)

        _compare(run, torch.float32, ("attention",), tol32=1e-4)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_scaled_pair_rows_and_plain_add(dtype):
    from fasttalk_llm_microservice_amd.ops import mixers as M

    g = torch.Generator().manual_seed(12)
    for T, n, H, dv in ((1, 7, 1, 3), (5, 300, 3, 72), (9, 64, 4, 128)):
        a, o = torch.randn(T, n, generator=g), torch.randn(T, H * dv, generator=g)
        wide = torch.randn(T, H * dv + 5, generator=g).to(dtype)
        _compare(lambda dev: (M.scaled_pair_rows(a.to(dev), 1.3, o.to(dev), wide.to(dev)[:, 5:], -0.4, 1e-5, H, dv, dtype),),
                 dtype, ("rows",))
        x, y, w = torch.randn(T, n, generator=g), torch.randn(T, n, generator=g).to(dtype), torch.rand(n, generator=g)

        def add(dev):
            r = x.clone().to(dev)
            h, c = M.add_rms_norm_rows(r, y.to(dev), None, 1e-5, next_w=w.to(dev), out_dtype=dtype, want_cast=True)
            return r, h, c

        _compare(add, dtype, ("residual", "normed", "cast"))


def test_graph_replays_of_new_kernels():
    """Decode rows of both recurrences, the convolutions' in-place histories, the sink attention and
    the grouped router inside a captured graph: several replays with eager work between them
    give what the eager calls give."""
    from fasttalk_llm_microservice_amd.ops import mixers as M

    g = torch.Generator().manual_seed(4)
    H, G, dk, dv, page, taps = 4, 2, 16, 16, 8, 3
    n, nv, nq, nk = G * dk, H * dv, H * dk, G * dk
    seg, slot_map, _, nb = _segments("cuda", [1, 1, 1], [25, 9, 1], [0, 2, 1], page, pad=1)
    r = lambda *s: torch.randn(*s, generator=g).cuda()   # noqa: E731
    p1, p2, p3, a, b = r(3, 2 * n + nv), r(3, nq + nk + G * dv), r(3, H * (2 * dk + 2 * dv)), r(3, H), r(3, H)
    w1, w2, a_log, dt = r(2 * n + nv, taps), r(nq + nk + G * dv, taps), r(H), r(H)
    router, h = r(6, 40), r(3, 40)
    table = M.rope_table(64, 16, 100.0, device="cuda")
    spec = M.WindowSpec(H, G, dk, dv, 6, 0.25, sink=r(H))
    ld = torch.log(torch.tensor([0.9, 0.99, 0.999, 1.0], dtype=torch.float64)).cuda()
    state0 = [r(3, taps - 1, 2 * n + nv), r(3, taps - 1, nq + nk + G * dv), r(3, H, dk, dv), r(3, H, dk, dv),
              r(nb, page, nk), r(nb, page, G * dv)]
    st = [t.clone() for t in state0]

    def step():
        q, k, v, lg, beta = M.conv_delta_prep(p1, a, b, w1, st[0], a_log, dt, seg, H, G, dk, dv)
        o1 = M.head_delta_rule(q, k, v, lg, beta, st[2], seg)
        q2 = M.conv_attn_prep(p2, nq, nk, w2, st[1], seg, None, None, 1e-5, dk, slot_map, st[4], st[5], table, 16, True)
        o2 = M.window_attention(q2, st[4], st[5], seg, spec)
        o3 = M.retention(p3, table, 16, ld, st[3], seg, H, dk, dv)
        y = M.scaled_pair_rows(o2.view(3, -1), 0.7, o3, p3[:, H * (2 * dk + dv):], 0.4, 1e-5, H, dv, torch.float32)
        idx, wts = M.moe_route_top_logits(h, router, None, 2, True, 1.5, 3, 2)
        return o1, y, idx, wts

    def reset():
        for t, t0 in zip(st, state0):
            t.copy_(t0)

    want = [t.clone() for t in step()]
    want_st = [t.clone() for t in st]
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
        for got, w in list(zip(out, want)) + list(zip(st, want_st)):
            torch.testing.assert_close(got, w, rtol=1e-6, atol=1e-6)
        _ = (torch.randn(64, 64, device="cuda") @ torch.randn(64, 64, device="cuda")).sum().item()
