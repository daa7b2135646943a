"""Shared cases of the Logirax tests: small configurations with random weights, run
through the framework's engine (scheduler, block / state-slot pools, model runner,
kernels or the CPU backend) and compared with tests/logirax_oracle.py.

None of the configurations is a real model's; they vary what a single model would leave
equal or 1: heads vs kv heads, one head, more heads than one matrix tile of the score mix
holds, key sizes over 64, windows of one page, one page + 1, a single position, longer than
the prompt; kept first tokens none / fewer / more than a window; rotary dims none / part /
all of a head; latent ranks of q and kv that differ either way, value sizes over 64 and
smaller than keys; one expert per token, every expert, with and without a shared expert of
another size; router, embedding and logit factors of 1; either mixer type first and last;
layers without feed-forward; widths that are no multiple of 4."""
import copy
import os
import sys

import torch

sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))
import logirax_oracle as O  # noqa: E402

from fasttalk_llm_microservice_amd.engine.config import EngineConfig  # noqa: E402
from fasttalk_llm_microservice_amd.engine.engine import LLMEngine  # noqa: E402
from fasttalk_llm_microservice_amd.models import logirax as L  # noqa: E402


def _att(heads, kv, dim, window, keep, scale, cap, rot=None):
    d = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": dim, "scale": scale, "softcap": cap,
         "mask": {"size": window, "keep_first": keep}}
    if rot:
        d["rot"] = {"dims": rot[0], "base": rot[1]}
    return d


def _lat(heads, dim, rot_dim, vdim, kv_rank, q_rank, scale, base=1000.0):
    return {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "q_rank": q_rank,
            "scale": scale, "rot": {"dims": rot_dim, "base": base}}


def _dense(ff, limit):
    return {"kind": "dense", "ff": ff, "limit": limit}


def _moe(experts, top, scale, ff, shared):
    d = {"kind": "moe", "router": {"experts": experts, "top": top, "scale": scale}, "expert": {"ff": ff}}
    if shared:
        d["shared"] = {"ff": shared}
    return d


def _layer(mixer, mlp):
    return {"type": "latent_attention" if "kv_rank" in mixer else "attention", "mixer": mixer, "mlp": mlp}


def _cfg(vocab, width, eps, scale, logit, layers):
    return {"architecture": "Logirax", "vocab": vocab, "width": width, "norm": {"eps": eps},
            "embedding": {"scale": scale}, "logit_scale": logit, "layers": layers}


CONFIGS = {
    # attention first; a window of one page + 1 with fewer kept tokens; part of each head rotated; kv heads =
    # heads once; a layer without feed-forward; a dense layer in the middle; latent attention last
    "a": _cfg(101, 64, 1e-5, 3.0, 1.5, [
        _layer(_att(4, 2, 12, 17, 3, 0.4, 5.0, (8, 100.0)), _moe(5, 2, 1.3, 24, 40)),
        _layer(_lat(3, 10, 8, 14, 20, 12, 0.3), _dense(48, 0.8)),
        _layer(_att(5, 5, 8, 9, 11, 0.7, 8.0, (8, 500.0)), None),
        _layer(_lat(2, 16, 4, 8, 9, 24, 0.25, 50.0), _moe(4, 1, 2.0, 32, 16)),
    ]),
    # latent attention first, with a value size over 64; a width that is no multiple of 4; one head; a window of
    # one position with kept tokens, no rotation; no shared expert; factors of 1
    "b": _cfg(77, 50, 1e-6, 1.0, 1.0, [
        _layer(_lat(2, 6, 2, 72, 33, 7, 0.4), None),
        _layer(_att(1, 1, 10, 1, 4, 0.5, 3.0), _moe(3, 3, 1.0, 20, 0)),
        _layer(_att(6, 2, 7, 1000, 0, 0.6, 20.0, (4, 50.0)), _moe(6, 2, 1.0, 12, 30)),
    ]),
    # 18 heads (two tiles of the score mix), a key size over 64, a window of exactly one page without kept
    # tokens, a small window with everything kept
    "c": _cfg(64, 40, 1e-5, 6.0, 0.5, [
        _layer(_att(18, 6, 8, 16, 0, 0.5, 10.0, (6, 10000.0)), _dense(28, 2.5)),
        _layer(_att(3, 1, 80, 4, 64, 0.15, 6.0, (80, 100.0)), _moe(9, 4, 0.7, 16, 8)),
        _layer(_lat(4, 8, 16, 8, 40, 40, 0.2, 10000.0), _moe(2, 1, 1.5, 20, 20)),
    ]),
}


def make_model(name, seed, tmp_path, tweak=None):
    """(checkpoint dir, config dict, fp32 tensors of the bf16 weights)."""
    cfg = copy.deepcopy(CONFIGS[name])
    lcfg = L.config_from_dict(cfg, name)
    t = L.random_tensors(lcfg, seed, torch.bfloat16)
    if tweak:
        tweak(t)
    d = os.path.join(str(tmp_path), f"{name}-{seed}")
    L.save_checkpoint(lcfg, t, d)
    return d, cfg, {k: v.float() for k, v in t.items()}


def make_engine(ckpt, device, dtype="float32", pages=64, seqs=4, page=16, graphs=False):
    """``graphs``: decode steps replay captured graphs and are queued ahead (the
    serving configuration on a GPU); otherwise every step runs eagerly."""
    return LLMEngine(EngineConfig(model=ckpt, weights=ckpt, device=device, dtype=dtype, num_kv_blocks=pages,
                                  block_size=page, max_num_seqs=seqs, max_model_len=pages * page,
                                  max_num_batched_tokens=pages * page, enforce_eager=not graphs,
                                  async_output=graphs, swap_space_gb=0.0))


def tokens(n, vocab, seed):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, vocab, (n,), generator=g).tolist()


def replay(eng, reqs, schedule):
    """reqs: id -> tokens.  schedule: steps, each a list of (id, count).  Every position's
    logits are asked for.  Returns id -> [T, vocab] tensor."""
    at = {i: 0 for i in reqs}
    rows = {i: [] for i in reqs}
    for step in schedule:
        entries, end = [], []
        for i, n in step:
            lo, hi = at[i], at[i] + n
            entries.append((i, reqs[i][lo:hi], list(range(n))))
            at[i] = hi
            if hi == len(reqs[i]):
                end.append(i)
        lg = torch.from_numpy(eng.replay_step(entries, end).copy())
        k = 0
        for i, n in step:
            rows[i].append(lg[k:k + n])
            k += n
    return {i: torch.cat(v) for i, v in rows.items()}


def close(got, want, dtype="float32"):
    if dtype == "float32":
        torch.testing.assert_close(got, want, rtol=3e-4, atol=4e-4)
        return
    # bf16: rounding differs from the oracle's everywhere, and a router's close call may go the
    # other way at single positions (the fp32 runs are the sharp ones)
    err = (got - want).pow(2).mean(-1).sqrt() / want.pow(2).mean(-1).sqrt().clamp_min(1e-3)
    assert err.median() < 0.06 and float((err > 0.25).float().mean()) <= 0.1, err


def oracle(cfg, P, toks):
    return O.forward(cfg, P, toks).float()


def portions(total, sizes):
    out, k = [], 0
    while total > 0:
        n = min(sizes[k % len(sizes)], total)
        out.append(n)
        total -= n
        k += 1
    return out
