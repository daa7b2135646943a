"""Pitelorn through the engine on the CPU backend (fp32) against the plain oracle, and
each mechanism of models/mixers.py alone against the oracle's function for it."""
import os
import sys

import pytest
import torch

sys.path.insert(0, os.path.dirname(os.path.dirname(os.path.abspath(__file__))))
import pitelorn_cases as C  # noqa: E402
import pitelorn_engine_cases as E  # noqa: E402
import pitelorn_mechanism_cases as K  # noqa: E402


@pytest.mark.parametrize("name", ["a", "b", "c"])
def test_whole_prompt(name, tmp_path):
    E.whole_prompt(name, "cpu", "float32", tmp_path)


@pytest.mark.parametrize("name", ["a", "b", "c"])
def test_layers(name, tmp_path):
    E.layers_of_a_prompt(name, "cpu", "float32", tmp_path)


@pytest.mark.parametrize("name", ["a", "b", "c"])
def test_prefill_then_decode(name, tmp_path):
    E.prefill_then_decode(name, "cpu", "float32", tmp_path)


@pytest.mark.parametrize("name", ["a", "c"])
def test_portions(name, tmp_path):
    E.portions_of_a_prompt(name, "cpu", "float32", tmp_path)


@pytest.mark.parametrize("name", ["a", "b", "c"])
def test_mixed_batches_and_reuse(name, tmp_path):
    E.mixed_batches_and_reuse(name, "cpu", "float32", tmp_path)


def test_peaked_scores(tmp_path):
    E.peaked_scores("cpu", "float32", tmp_path)


def test_raised_and_lowered_sinks(tmp_path):
    E.raised_and_lowered_sinks("cpu", "float32", tmp_path)


def test_slow_decay_long_decode(tmp_path):
    E.slow_decay_long_decode("cpu", "float32", tmp_path)


@pytest.mark.parametrize("name", ["a", "b"])
def test_greedy_generation(name, tmp_path):
    E.greedy_generation(name, "cpu", "float32", tmp_path)


@pytest.mark.parametrize("case", K.CASES)
def test_mechanism(case):
    K.run(case, "cpu", torch.float32)


def test_registry_and_config(tmp_path):
    from fasttalk_llm_microservice_amd.models import pitelorn as PT
    from fasttalk_llm_microservice_amd.models.config import resolve_model
    from fasttalk_llm_microservice_amd.models.registry import architecture_of

    d, cfg, _ = C.make_model("a", 1, tmp_path)
    mc = resolve_model(d)
    assert architecture_of(mc).name == "pitelorn" and mc.vocab_size == cfg["vocab"]
    assert [r[0] for r in mc.runs()] == [0, 1, 2, 3] and mc.layers[2]["mlp"] is None
    assert mc.bigram == (37, 5, 3) and mc.layers[3]["mixer"]["right_scale"] == -0.8
    assert mc.layers[1]["mlp"]["router"]["groups"] == {"count": 3, "keep": 2}
    assert architecture_of(resolve_model("pitelorn-tiny")).name == "pitelorn"
    assert architecture_of(resolve_model("logirax-tiny")).name == "logirax"
    assert architecture_of(resolve_model("tiny")).name == "llama"
    # the written configuration parses back to itself; what the design does not have is refused
    assert PT.config_from_dict(PT.config_to_dict(mc), mc.name) == mc
    delta, par = cfg["layers"][0], cfg["layers"][1]
    right = {**par["mixer"]["right"], "decay": [0.9]}
    for bad in ({**delta, "type": "mamba2"}, {**delta, "mlp": {"kind": "gelu", "ff": 8}},
                {**par, "mixer": {**par["mixer"], "right": right}}):
        with pytest.raises(ValueError):
            PT.config_from_dict({**cfg, "layers": [bad]})


def test_cache_and_state_per_layer(tmp_path):
    """Delta layers own an fp32 state and the convolution's last inputs per slot; side-by-side
    layers own paged keys and values, the convolution's last inputs and an fp32 state; the
    previous token has one entry per slot."""
    d, cfg, _ = C.make_model("a", 2, tmp_path)
    eng = C.make_engine(d, "cpu", pages=8, seqs=3)
    kv = eng.runner.kv
    assert len(kv.per_run) == 4 and kv.extra["last_token"].shape == (3,)
    m = cfg["layers"][0]["mixer"]
    st, hist = kv.per_run[0]
    assert st.shape == (3, m["heads"], m["dim"], m["vdim"]) and st.dtype == torch.float32
    assert hist.shape == (3, m["conv"] - 1, 2 * m["kv_heads"] * m["dim"] + m["heads"] * m["vdim"])
    (kc, vc, hist), st = kv.per_run[1]
    a, b = cfg["layers"][1]["mixer"]["left"], cfg["layers"][1]["mixer"]["right"]
    assert kc.shape == (8, 16, a["kv_heads"] * a["dim"]) and vc.shape == (8, 16, a["kv_heads"] * a["vdim"])
    assert hist.shape[1:] == (a["conv"] - 1, a["heads"] * a["dim"] + a["kv_heads"] * (a["dim"] + a["vdim"]))
    assert st.shape == (3, b["heads"], b["dim"], b["vdim"]) and st.dtype == hist.dtype == torch.float32
    model = eng.runner.model
    assert model.kv_bytes_per_token(4) == model.cfg.kv_bytes_per_token(4)
    assert model.head is not None and model.resident_weight_bytes() > 0
