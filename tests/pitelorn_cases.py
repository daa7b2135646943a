"""Shared cases of the Pitelorn tests: small configurations with random weights, run
through the framework's engine (scheduler, block / state-slot pools, model runner,
kernels or the CPU backend) and compared with tests/pitelorn_oracle.py.

None of the configurations is a real model's; they vary what a single model would leave
equal or 1: heads vs kv heads, one head; key vs value sizes, sizes that are no multiple of
4 / 16 / 64, key sizes over 64 and over 128, value sizes over 64; convolutions of 1 to 5
taps, different ones in the two mixers; windows of one position, one page, one page + 1,
longer than the prompt; rotary dims none / part / all of a head, with and without the
ramp; decays near 1, of exactly 1 and small; side-by-side scales of 1, of 0.3 and negative;
expert groups of several, of one expert, a single group, every group kept, every expert
chosen; router scale 1; no pair table; either mixer type first and last; layers without
feed-forward; a width that is no multiple of 4."""
import copy
import os
import sys

import torch

sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))
import pitelorn_oracle as O  # noqa: E402
from logirax_cases import make_engine, portions, replay, tokens  # noqa: E402,F401

from fasttalk_llm_microservice_amd.models import pitelorn as PT  # noqa: E402


def _delta(heads, kv, dim, vdim, taps):
    return {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "conv": taps}


def _rot(dims, base, scaling=None):
    d = {"dims": dims, "base": base}
    if scaling:
        d["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    return d


def _par(heads, kv, dim, vdim, window, taps, scale, rot, rh, rdim, rvdim, decay, rrot, scales):
    left = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "conv": taps, "scale": scale,
            "mask": {"size": window}}
    right = {"heads": rh, "dim": rdim, "vdim": rvdim, "decay": decay}
    if rot:
        left["rot"] = rot
    if rrot:
        right["rot"] = rrot
    return {"left": left, "right": right, "left_scale": scales[0], "right_scale": scales[1]}


def _dense(ff):
    return {"kind": "dense", "ff": ff}


def _moe(experts, top, scale, groups, keep, ff, limit):
    return {"kind": "moe", "router": {"experts": experts, "top": top, "scale": scale,
                                      "groups": {"count": groups, "keep": keep}}, "expert": {"ff": ff, "limit": limit}}


def _layer(mixer, mlp):
    return {"type": "parallel" if "left" in mixer else "delta", "mixer": mixer, "mlp": mlp}


def _cfg(vocab, width, eps, bigram, layers):
    e = {"bigram": dict(zip(("buckets", "mul_prev", "mul_cur"), bigram))} if bigram else {}
    return {"architecture": "Pitelorn", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": e,
            "layers": layers}


CONFIGS = {
    # delta first; a window of one page + 1; part of each head rotated with the ramp; several expert
    # groups; a layer without feed-forward in the middle
    "a": _cfg(101, 64, 1e-5, (37, 5, 3), [
        _layer(_delta(4, 2, 12, 20, 4), _dense(48)),
        _layer(_par(4, 2, 12, 8, 17, 3, 0.3, _rot(8, 1000.0, (4.0, 64, 4.0, 1.0)), 3, 10, 24, [0.9, 0.99, 0.999],
                    _rot(6, 100.0), (1.1, 0.3)), _moe(6, 2, 1.7, 3, 2, 24, 0.9)),
        _layer(_delta(3, 3, 16, 16, 2), None),
        _layer(_par(2, 2, 16, 16, 33, 5, 0.25, _rot(16, 500.0), 2, 32, 40, [0.5, 0.97], _rot(32, 5000.0),
                    (0.6, -0.8)), _moe(8, 3, 1.0, 2, 1, 16, 3.0)),
    ]),
    # side by side first; no pair table; one-tap convolutions; no rotation; a window of one position; a
    # decay of 1; value sizes over 64; every expert chosen of one group; a width of 50
    "b": _cfg(77, 50, 1e-6, None, [
        _layer(_par(2, 2, 6, 72, 1, 1, 0.4, None, 1, 72, 33, [1.0], None, (1.0, 1.0)), None),
        _layer(_delta(2, 1, 33, 7, 1), _moe(3, 3, 1.0, 1, 1, 20, 0.5)),
        _layer(_par(3, 1, 7, 5, 1000, 2, 0.5, _rot(4, 50.0, (2.0, 16, 2.0, 0.5)), 4, 9, 6, [0.8, 0.9, 0.95, 0.99],
                    _rot(2, 20.0), (0.9, 1.2)), _dense(20)),
    ]),
    # key sizes over 64 and over 128; a window of exactly one page; groups of one expert each; all groups kept
    "c": _cfg(64, 40, 1e-5, (7, 2, 9), [
        _layer(_par(3, 1, 80, 16, 16, 4, 0.1, _rot(80, 10000.0, (8.0, 32, 8.0, 2.0)), 2, 128, 132, [0.98, 0.9995],
                    _rot(64, 10000.0), (0.7, 0.5)), _moe(5, 2, 2.0, 5, 3, 28, 1.5)),
        _layer(_delta(6, 2, 136, 8, 3), _moe(4, 1, 0.7, 2, 2, 12, 8.0)),
        _layer(_delta(2, 2, 68, 80, 4), _dense(16)),
    ]),
}


def make_model(name, seed, tmp_path, tweak=None, dtype="float32"):
    """(checkpoint dir, config dict, fp32 tensors of the bf16 weights).  For bf16 runs the routers
    choose every expert: with random weights a choice is often close, and one that rounding
    turns over moves the logits by as much as a fault would."""
    cfg = copy.deepcopy(CONFIGS[name])
    if dtype != "float32":
        for l in cfg["layers"]:
            if l["mlp"] and l["mlp"]["kind"] == "moe":
                r = l["mlp"]["router"]
                r["top"], r["groups"]["keep"] = r["experts"], r["groups"]["count"]
    pcfg = PT.config_from_dict(cfg, name)
    t = PT.random_tensors(pcfg, seed, torch.bfloat16)
    if tweak:
        tweak(t)
    d = os.path.join(str(tmp_path), f"{name}-{seed}")
    PT.save_checkpoint(pcfg, t, d)
    return d, cfg, {k: v.float() for k, v in t.items()}


def close(got, want, dtype="float32"):
    if dtype == "float32":
        torch.testing.assert_close(got, want, rtol=3e-4, atol=4e-4)
        return
    # bf16: rounding differs from the oracle's everywhere (the fp32 runs are the sharp ones)
    err = (got - want).pow(2).mean(-1).sqrt() / want.pow(2).mean(-1).sqrt().clamp_min(1e-3)
    assert err.median() < 0.06 and float(err.max()) < 0.25, err


def oracle(cfg, P, toks):
    return O.forward(cfg, P, toks).float()
