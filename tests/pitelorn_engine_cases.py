"""Engine-level Pitelorn cases, run by tests/unit/test_pitelorn_cpu.py (CPU backend) and
tests/test_pitelorn_gpu.py (HIP kernels) with the device and dtype as arguments."""
import torch

import pitelorn_cases as C
import pitelorn_oracle as O

from fasttalk_llm_microservice_amd.engine.sampling_params import SamplingParams


def whole_prompt(name, device, dtype, tmp):
    d, cfg, P = C.make_model(name, 11, tmp, dtype=dtype)
    eng = C.make_engine(d, device, dtype)
    for n, seed in ((1, 1), (2, 2), (3, 3), (37, 4), (130, 5)):   # the first tokens, then one and several chunks
        t = C.tokens(n, cfg["vocab"], seed)
        got = C.replay(eng, {"r": t}, [[("r", n)]])["r"]
        C.close(got, C.oracle(cfg, P, t), dtype)


def layers_of_a_prompt(name, device, dtype, tmp):
    """The residual after every layer against the oracle's."""
    d, cfg, P = C.make_model(name, 18, tmp, dtype=dtype)
    eng = C.make_engine(d, device, dtype)
    t = C.tokens(70, cfg["vocab"], 6)
    eng.runner.model.layer_tap = tap = []
    C.replay(eng, {"r": t}, [[("r", len(t))]])
    eng.runner.model.layer_tap = None
    want = O.layers(cfg, P, t)
    assert len(tap) == len(want)
    for g, w in zip(tap, want):
        torch.testing.assert_close(g.float().cpu(), w.float(), rtol=3e-4, atol=3e-4)


def prefill_then_decode(name, device, dtype, tmp):
    """Windows pass over decoded tokens; the previous token, the convolutions' last inputs and
    both recurrences' states come from the step before."""
    d, cfg, P = C.make_model(name, 12, tmp, dtype=dtype)
    eng = C.make_engine(d, device, dtype)
    for first in (1, 2, 19, 40):
        t = C.tokens(first + 40, cfg["vocab"], 5 + first)
        sched = [[("r", first)]] + [[("r", 1)]] * 40
        C.close(C.replay(eng, {"r": t}, sched)["r"], C.oracle(cfg, P, t), dtype)


def portions_of_a_prompt(name, device, dtype, tmp):
    d, cfg, P = C.make_model(name, 13, tmp, dtype=dtype)
    eng = C.make_engine(d, device, dtype)
    t = C.tokens(150, cfg["vocab"], 9)
    want = C.oracle(cfg, P, t)
    # page size 16: cuts on and off page and window borders; 32+ rows take the chunk form of the
    # recurrences (chunks of 64 rows) and the matrix-product attention, more than 64 the sorted
    # experts, fewer the row walks, the per-row attention and the per-pair experts
    for sizes in ((2,), (1, 1, 1, 2, 3), (3, 2, 16, 1, 17, 5), (31, 32, 33), (64, 2), (33, 41, 1, 40), (65, 63, 22),
                  (100, 50)):
        sched = [[("r", n)] for n in C.portions(len(t), sizes)]
        C.close(C.replay(eng, {"r": t}, sched)["r"], want, dtype)


def mixed_batches_and_reuse(name, device, dtype, tmp):
    """Unequal requests side by side (portions beside single tokens), more requests
    than state slots over time, a page pool smaller than the sum of all requests."""
    d, cfg, P = C.make_model(name, 14, tmp, dtype=dtype)
    eng = C.make_engine(d, device, dtype, pages=12, seqs=3)          # 192 tokens of cache, 3 slots
    lens = {"a": 110, "b": 9, "c": 41, "d": 1, "e": 55, "f": 40}
    reqs = {i: C.tokens(n, cfg["vocab"], 20 + k) for k, (i, n) in enumerate(lens.items())}
    sched = [
        [("a", 17), ("b", 1)],
        [("b", 1), ("a", 70), ("c", 5)],
        [("a", 1), ("b", 7), ("c", 1)],            # b ends: its slot and pages go back
        [("c", 33), ("a", 1), ("d", 1)],           # d takes b's slot; d ends
        [("a", 21), ("c", 1)],                     # a ends
        [("c", 1), ("e", 2), ("f", 36)],           # e, f reuse a's and d's slots and pages; c ends
        [("f", 1), ("e", 50)],
        [("e", 1), ("f", 3)],
        [("e", 1)],
        [("e", 1)],
    ]
    got = C.replay(eng, reqs, sched)
    for i, t in reqs.items():
        C.close(got[i], C.oracle(cfg, P, t), dtype)
    assert eng.scheduler.slots.num_free() == 3 and eng.bm.num_free() == 12
    # the same requests alone, one whole step each, give the same logits as in the batch
    if dtype == "float32":
        for i in ("a", "e"):
            alone = C.replay(eng, {i: reqs[i]}, [[(i, len(reqs[i]))]])[i]
            torch.testing.assert_close(alone, got[i], rtol=3e-4, atol=4e-4)


def peaked_scores(device, dtype, tmp):
    """Query projections scaled up: each row's weight sits on few keys anywhere in its window (at
    its edge, at page borders), so a key lost or seen one position too far shows."""
    def tweak(t):
        for k in t:
            if k.endswith("left.q"):
                t[k] *= 6.0
    for name in ("a", "c"):
        d, cfg, P = C.make_model(name, 15, tmp, tweak, dtype)
        eng = C.make_engine(d, device, dtype, pages=24)
        t = C.tokens(200, cfg["vocab"], 31)
        want = C.oracle(cfg, P, t)
        C.close(C.replay(eng, {"r": t}, [[("r", 150)]] + [[("r", 1)]] * 50)["r"], want, dtype)
        sched = [[("r", n)] for n in C.portions(200, (15, 17, 16, 1, 31, 33, 2, 100))]
        C.close(C.replay(eng, {"r": t}, sched)["r"], want, dtype)


def raised_and_lowered_sinks(device, dtype, tmp):
    """Sinks that take most of a row's weight in one head and none in the next."""
    def tweak(t):
        for k in t:
            if k.endswith("sink"):
                t[k] = torch.tensor([3.0 if i % 2 else -9.0 for i in range(t[k].numel())]).bfloat16()
    for name in ("a", "b"):
        d, cfg, P = C.make_model(name, 19, tmp, tweak, dtype)
        eng = C.make_engine(d, device, dtype)
        t = C.tokens(60, cfg["vocab"], 33)
        C.close(C.replay(eng, {"r": t}, [[("r", 34)], [("r", 6)]] + [[("r", 1)]] * 20)["r"], C.oracle(cfg, P, t), dtype)


def slow_decay_long_decode(device, dtype, tmp):
    """Delta-rule decays near 1 beside retention decays near 1: 120 single-token steps after a
    three-token prompt carry both states (and the convolutions, the previous token, the caches)
    through every step; a state that is lost or reset shows."""
    def tweak(t):
        for k in t:
            if k.endswith("A_log"):
                t[k] -= 3.0
    d, cfg, P = C.make_model("c", 16, tmp, tweak, dtype)
    eng = C.make_engine(d, device, dtype)
    t = C.tokens(123, cfg["vocab"], 41)
    C.close(C.replay(eng, {"r": t}, [[("r", 3)]] + [[("r", 1)]] * 120)["r"], C.oracle(cfg, P, t), dtype)


def greedy_generation(name, device, dtype, tmp, graphs=False):
    """Through LLMEngine.generate: the scheduler's own batching, the sampler at
    temperature 0, against greedy decoding with the oracle."""
    d, cfg, P = C.make_model(name, 17, tmp, dtype=dtype)
    eng = C.make_engine(d, device, dtype, seqs=2, graphs=graphs)   # three prompts, two slots: one waits
    prompts = [C.tokens(n, cfg["vocab"], 50 + n) for n in (5, 1, 40)]
    outs = eng.generate(prompts, SamplingParams(temperature=0.0, max_tokens=9, ignore_eos=True))
    for p, out in zip(prompts, outs):
        assert len(out) == 9
        lg = O.forward(cfg, P, list(p) + list(out))
        for k, tok in enumerate(out):
            row = lg[len(p) - 1 + k]
            best = int(row.argmax())
            if best != tok:   # only a near-tie may differ
                assert row[best] - row[tok] < 1e-3, (p, k, tok, best)
    assert eng.scheduler.slots.num_free() == 2
    if graphs:
        assert eng.runner.stats["graph_replays"] > 0
