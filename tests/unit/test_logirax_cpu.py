"""Logirax through the engine on the CPU backend (fp32) against the plain oracle, and
each mechanism of models/mixers.py alone against the oracle's function for it."""
import os
import sys

import pytest
import torch

sys.path.insert(0, os.path.dirname(os.path.dirname(os.path.abspath(__file__))))
import logirax_cases as C  # noqa: E402
import logirax_engine_cases as E  # noqa: E402
import logirax_mechanism_cases as K  # noqa: E402


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


def test_shifted_long_decode(tmp_path):
    E.shifted_long_decode("cpu", "float32", tmp_path)


@pytest.mark.parametrize("name", ["a", "b"])
def test_greedy_generation(name, tmp_path):
    E.greedy_generation(name, "cpu", "float32", tmp_path)


@pytest.mark.parametrize("case", K.CASES)
def test_mechanism(case):
    K.run(case, "cpu", torch.float32)


def test_registry_and_config(tmp_path):
    from fasttalk_llm_microservice_amd.models import logirax as LX
    from fasttalk_llm_microservice_amd.models.config import resolve_model
    from fasttalk_llm_microservice_amd.models.registry import architecture_of

    d, cfg, _ = C.make_model("a", 1, tmp_path)
    mc = resolve_model(d)
    assert architecture_of(mc).name == "logirax" and mc.vocab_size == cfg["vocab"]
    assert [r[0] for r in mc.runs()] == [0, 1, 2, 3] and mc.layers[2]["mlp"] is None
    assert mc.embed_scale == 3.0 and mc.logit_scale == 1.5 and mc.layers[3]["mlp"]["router"]["scale"] == 2.0
    assert architecture_of(resolve_model("logirax-tiny")).name == "logirax"
    assert architecture_of(resolve_model("nulazen-tiny")).name == "nulazen"
    assert architecture_of(resolve_model("tiny")).name == "llama"
    # the written configuration parses back to itself; what the design does not have is refused
    assert LX.config_from_dict(LX.config_to_dict(mc), mc.name) == mc
    att, lat = cfg["layers"][0], cfg["layers"][1]
    for bad in ({**att, "type": "mamba2"}, {**att, "mixer": {**att["mixer"], "vdim": 5}},
                {**lat, "mixer": {**lat["mixer"], "rot": {"dims": 2, "base": 10.0}}},
                {**att, "mlp": {"kind": "gelu", "ff": 8}}):
        with pytest.raises(ValueError):
            LX.config_from_dict({**cfg, "layers": [bad]})


def test_cache_and_state_per_layer(tmp_path):
    """Attention layers own paged keys and values (both of the key's size), latent layers one
    paged row of latent and rotated part, and every layer an fp32 input row per slot."""
    d, cfg, _ = C.make_model("a", 2, tmp_path)
    eng = C.make_engine(d, "cpu", pages=8, seqs=3)
    kv = eng.runner.kv
    a, l = cfg["layers"][0]["mixer"], cfg["layers"][1]["mixer"]
    assert len(kv.per_run) == 4
    assert [t.shape for t in kv.per_run[0]] == [(8, 16, a["kv_heads"] * a["dim"])] * 2
    assert kv.per_run[1].shape == (8, 16, l["kv_rank"] + l["rot_dim"])
    assert [t.shape for t in kv.extra["prev_h"]] == [(3, cfg["width"])] * 4
    assert all(t.dtype == torch.float32 for t in kv.extra["prev_h"])
    model = eng.runner.model
    assert model.kv_bytes_per_token(4) == model.cfg.kv_bytes_per_token(4)
    assert model.head is not None and model.resident_weight_bytes() > 0
