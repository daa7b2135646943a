"""Pitelorn: a decoder-only model with a norm in front of each sublayer (weights stored as
offsets from one, x / rms(x) * (1 + w)) and no norm behind it: x += mixer(norm1 x);
x += ff(norm2 x).

* Embedding: embed[token] plus a row of the pair table ``bigram``, chosen by (previous token *
  mul_prev + token * mul_cur) mod buckets; a sequence's first token takes row ``buckets``.
  The previous token lives in the sequence's state slot.
* Mixer ``delta``: the gated delta rule with one decay per head behind short convolutions
  (:class:`..models.mixers.HeadDelta`).
* Mixer ``parallel``: left_scale * left + right_scale * right on the same input
  (:class:`..models.mixers.SideBySideSum`) -- ``left``: windowed attention with convolved q, k
  and v, rotated pairs of neighbours (frequencies ramped down for long contexts) and a
  learned sink per head (:class:`..models.mixers.ConvSinkAttention`); ``right``: retention
  with a fixed decay per head (:class:`..models.mixers.Retention`).
* Feed-forward (optional per layer): dense down(silu(gate h) * (up h)), or clamped-GLU experts
  chosen by sigmoid scores within the best groups (:class:`..models.mixers.MoEFF`).
* Output: the model's norm, then ``head``.

Every size comes from ``config.json`` (keys: vocab, width, norm.eps, embedding.bigram{buckets,
mul_prev, mul_cur}, layers[].type / mixer / mlp{kind dense: ff; kind moe: router{experts, top,
scale, groups{count, keep}}, expert{ff, limit}}) or from tensor shapes.  Tensor names: embed,
bigram, head, final.norm, l<i>.{norm1,norm2},
l<i>.mix.{q,k,v,q.conv,k.conv,v.conv,a,b,g,A_log,dt_bias,norm,o},
l<i>.mix.left.{q,k,v,q.conv,k.conv,v.conv,sink,o}, l<i>.mix.right.{q,k,v,g,o},
l<i>.mlp.{gate,up,down}, l<i>.mlp.{router,e<j>.gate,e<j>.up,e<j>.down}.

The model body (layer runs, residual, caches, logits) is :class:`..models.stacked.StackedModel`.
"""
from __future__ import annotations

import dataclasses
import json
import os
from typing import Dict, List, Optional, Tuple

import torch

from .mixers import ConvSinkAttention, GatedFF, HeadDelta, MoEFF, Retention, SideBySideSum
from .registry import Architecture, register
from .stacked import StackedLayer, StackedModel

DELTA, PARALLEL = "delta", "parallel"


@dataclasses.dataclass(frozen=True)
class PitelornConfig:
    name: str
    vocab_size: int
    hidden_size: int
    rms_norm_eps: float
    bigram: Optional[tuple]            # (buckets, mul_prev, mul_cur) or None
    layers: tuple                      # per layer: dict(type=, mixer=, mlp=)
    max_position_embeddings: int = 1 << 17
    bos_token_id: int = 0
    eos_token_ids: tuple = ()
    tie_word_embeddings: bool = False
    architecture = "pitelorn"

    @property
    def num_layers(self) -> int:
        return len(self.layers)

    def runs(self) -> List[Tuple[int, Optional[int]]]:
        return [(i, None) for i in range(len(self.layers))]

    def num_params(self) -> int:
        return sum(int(torch.Size(s).numel()) for s in tensor_shapes(self).values())

    def kv_bytes_per_token(self, dtype_bytes: int = 2) -> int:
        return sum(m["kv_heads"] * (m["dim"] + m["vdim"]) * dtype_bytes
                   for m in (l["mixer"]["left"] for l in self.layers if l["type"] == PARALLEL))


def _sizes(m: dict, *dflt) -> dict:
    """A mixer's entry with the sizes it may leave out: kv_heads = heads, vdim = dim."""
    m = dict(m)
    m.setdefault("vdim", m["dim"])
    if "kv_heads" in dflt:
        m.setdefault("kv_heads", m["heads"])
    return m


def _mlp(i: int, mlp: Optional[dict]) -> Optional[dict]:
    if mlp is None:
        return None
    kind = mlp.get("kind", "dense")
    if kind == "dense":
        return {"kind": "dense", "ff": int(mlp["ff"])}
    if kind != "moe":
        raise ValueError(f"layer {i}: unknown feed-forward kind {kind!r}")
    r = mlp["router"]
    g = r.get("groups") or {}
    return {"kind": "moe", "expert": {"ff": int(mlp["expert"]["ff"]), "limit": float(mlp["expert"]["limit"])},
            "router": {"experts": int(r["experts"]), "top": int(r["top"]), "scale": float(r.get("scale", 1.0)),
                       "groups": {"count": int(g.get("count", 1)), "keep": int(g.get("keep", g.get("count", 1)))}}}


def config_from_dict(c: dict, name: str = "pitelorn") -> PitelornConfig:
    layers = []
    for i, l in enumerate(c["layers"]):
        m = l["mixer"]
        if l["type"] == DELTA:
            m = _sizes(m, "kv_heads")
        elif l["type"] == PARALLEL:
            m = {"left": _sizes(m["left"], "kv_heads"), "right": _sizes(m["right"]),
                 "left_scale": float(m.get("left_scale", 1.0)), "right_scale": float(m.get("right_scale", 1.0))}
            if len(m["right"]["decay"]) != m["right"]["heads"]:
                raise ValueError(f"layer {i}: one decay per retention head")
        else:
            raise ValueError(f"layer {i}: unknown mixer type {l['type']!r}")
        layers.append({"type": l["type"], "mixer": m, "mlp": _mlp(i, l.get("mlp"))})
    bg = (c.get("embedding") or {}).get("bigram")
    return PitelornConfig(name=name, vocab_size=int(c["vocab"]), hidden_size=int(c["width"]),
                          rms_norm_eps=float(c.get("norm", {}).get("eps", 1e-6)),
                          bigram=(int(bg["buckets"]), int(bg["mul_prev"]), int(bg["mul_cur"])) if bg else None,
                          layers=tuple(layers), max_position_embeddings=int(c.get("max_positions", 1 << 17)))


def config_to_dict(cfg: PitelornConfig) -> dict:
    emb = {}
    if cfg.bigram:
        emb["bigram"] = {"buckets": cfg.bigram[0], "mul_prev": cfg.bigram[1], "mul_cur": cfg.bigram[2]}
    return {"architecture": "Pitelorn", "vocab": cfg.vocab_size, "width": cfg.hidden_size,
            "norm": {"eps": cfg.rms_norm_eps}, "embedding": emb,
            "layers": [json.loads(json.dumps(l)) for l in cfg.layers]}


def tensor_shapes(cfg: PitelornConfig) -> Dict[str, tuple]:
    """Names and shapes of a checkpoint of this configuration (random init, tests)."""
    w, v = cfg.hidden_size, cfg.vocab_size
    t: Dict[str, tuple] = {"embed": (v, w), "final.norm": (w,), "head": (v, w)}
    if cfg.bigram:
        t["bigram"] = (cfg.bigram[0] + 1, w)
    for i, l in enumerate(cfg.layers):
        p, m = f"l{i}.", l["mixer"]
        t[p + "norm1"] = (w,)
        if l["type"] == DELTA:
            h, g, dk, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
            q = p + "mix."
            t.update({q + "q": (g * dk, w), q + "k": (g * dk, w), q + "v": (h * dv, w), q + "g": (h * dv, w),
                      q + "a": (h, w), q + "b": (h, w), q + "A_log": (h,), q + "dt_bias": (h,), q + "norm": (dv,),
                      q + "o": (w, h * dv)})
            conv = (q, m["conv"], (g * dk, g * dk, h * dv))
        else:
            a, b = m["left"], m["right"]
            h, g, dk, dv = a["heads"], a["kv_heads"], a["dim"], a["vdim"]
            q, r = p + "mix.left.", p + "mix.right."
            t.update({q + "q": (h * dk, w), q + "k": (g * dk, w), q + "v": (g * dv, w), q + "sink": (h,),
                      q + "o": (w, h * dv)})
            conv = (q, a["conv"], (h * dk, g * dk, g * dv))
            h, dk, dv = b["heads"], b["dim"], b["vdim"]
            t.update({r + "q": (h * dk, w), r + "k": (h * dk, w), r + "v": (h * dv, w), r + "g": (h * dv, w),
                      r + "o": (w, h * dv)})
        for n, rows in zip("qkv", conv[2]):
            t[f"{conv[0]}{n}.conv"] = (rows, conv[1])
        f, q = l["mlp"], p + "mlp."
        if f is not None:
            t[p + "norm2"] = (w,)
            if f["kind"] == "dense":
                t.update({q + "gate": (f["ff"], w), q + "up": (f["ff"], w), q + "down": (w, f["ff"])})
            else:
                t[q + "router"] = (f["router"]["experts"], w)
                for e in range(f["router"]["experts"]):
                    ff = f["expert"]["ff"]
                    t.update({f"{q}e{e}.gate": (ff, w), f"{q}e{e}.up": (ff, w), f"{q}e{e}.down": (w, ff)})
    return t


def random_tensors(cfg: PitelornConfig, seed: int = 0, dtype=torch.bfloat16, device="cpu") -> Dict[str, torch.Tensor]:
    """Random weights of the configuration's shapes: projections ~ N(0, 1/fan_in), norm offsets
    near 0, plain norm weights near 1, convolutions that favour the current token, decays
    that keep the recurrence lively."""
    g = torch.Generator(device=device).manual_seed(seed)
    out: Dict[str, torch.Tensor] = {}
    for name, shape in tensor_shapes(cfg).items():
        leaf = name.split(".")[-1]
        r = torch.rand(shape, generator=g, device=device)
        n = torch.randn(shape, generator=g, device=device)
        if name in ("embed", "bigram"):
            x = n
        elif leaf == "conv":
            x = 0.3 * n
            x[:, -1] += 0.7
        elif len(shape) == 2:
            x = n * shape[1] ** -0.5
        elif leaf == "A_log":
            x = -2.0 + 2.0 * r
        elif leaf in ("dt_bias", "sink"):
            x = n
        elif leaf == "norm" and name != "final.norm":
            x = 0.75 + 0.5 * r
        else:                                    # offset norms
            x = 0.25 * (r - 0.5)
        out[name] = x.to(dtype)
    return out


def save_checkpoint(cfg: PitelornConfig, tensors: Dict[str, torch.Tensor], out_dir: str):
    from safetensors.torch import save_file

    os.makedirs(out_dir, exist_ok=True)
    save_file({k: v.contiguous().cpu() for k, v in tensors.items()}, os.path.join(out_dir, "model.safetensors"))
    with open(os.path.join(out_dir, "config.json"), "w") as f:
        json.dump(config_to_dict(cfg), f, indent=1)


class PitelornModel(StackedModel):
    family = "Pitelorn"
    # steps of more rows sort them by expert, which is not captured
    max_graph_rows = MoEFF.PAIR_ROWS

    def load_tensors(self, get, has=lambda n: True):
        cfg, dev, dt = self.cfg, self.device, self.dtype
        eps, width = cfg.rms_norm_eps, cfg.hidden_size
        self.load_head(get, has)
        self.final_norm = self.offset_norm_weight(get("final.norm"))
        if cfg.bigram:
            self.load_pair_table(get("bigram"), *cfg.bigram)
        max_pos = max(self.max_model_len, 16) + 1
        self.layers = []
        for i, l in enumerate(cfg.layers):
            p, m, f = f"l{i}.", l["mixer"], l["mlp"]
            under = lambda part, p=p: lambda n: get(p + part + n)   # noqa: E731
            if l["type"] == DELTA:
                mixer = HeadDelta(under("mix."), width, m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["conv"], eps,
                                  dt, dev)
            else:
                mixer = self._parallel(under, m, max_pos)
            L = StackedLayer(l["type"], self.offset_norm_weight(get(p + "norm1")), None, mixer)
            if f is not None:
                L.norm2 = self.offset_norm_weight(get(p + "norm2"))
                if f["kind"] == "dense":
                    L.ff = GatedFF(under("mlp."), dt, dev, act="silu")
                else:
                    r = f["router"]
                    L.ff = MoEFF(under("mlp."), r["experts"], r["top"], f["expert"]["limit"], r["groups"]["count"],
                                 r["groups"]["keep"], None, dt, dev, routing="top_sigmoid", act="clamp_glu",
                                 route_scale=r["scale"])
            self.layers.append(L)
        return self

    def _parallel(self, under, m: dict, max_pos: int) -> SideBySideSum:
        dt, dev, eps, width = self.dtype, self.device, self.cfg.rms_norm_eps, self.cfg.hidden_size
        a, b = m["left"], m["right"]
        rot, sc = a.get("rot") or {}, (a.get("rot") or {}).get("scaling")
        left = ConvSinkAttention(
            under("mix.left."), width, a["heads"], a["kv_heads"], a["dim"], a["vdim"], a["conv"], a["scale"], 0.0, eps,
            dt, dev, window=int((a.get("mask") or {}).get("size", 0)), sink="learned", qk_norm=False,
            rot_dims=int(rot.get("dims", 0)), rot_base=float(rot.get("base", 10000.0)),
            rot_ramp=(sc["factor"], sc["original"], sc["fast"], sc["slow"]) if sc else None, interleaved=True,
            max_pos=max_pos)
        rot = b.get("rot") or {}
        right = Retention(under("mix.right."), width, b["heads"], b["dim"], b["vdim"], b["decay"],
                          int(rot.get("dims", 0)), float(rot.get("base", 10000.0)), eps, dt, dev, max_pos)
        return SideBySideSum(left, right, m["left_scale"], m["right_scale"], dt, dev)

    def random_tensors(self, seed: int, device):
        return random_tensors(self.cfg, seed, torch.bfloat16, device=device)


# ---------------------------------------------------------------------------------------
# registry: shapes for random-init runs (benchmarks, smoke tests)
# ---------------------------------------------------------------------------------------

def _delta(heads, kv_heads, dim, vdim, taps):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": taps}


def _par(heads, kv_heads, dim, vdim, window, taps, ret_heads, ret_dim, ret_vdim, rot_dims=None, scaling=True):
    rot = {"dims": rot_dims or dim, "base": 500000.0}
    if scaling:
        rot["scaling"] = {"factor": 8.0, "original": 8192, "fast": 24.0, "slow": 2.0}
    # decays spaced evenly in log2(1 - d), from 1 - 2^-5 on
    decay = [1.0 - 2.0 ** (-5.0 - 5.0 * j / max(ret_heads - 1, 1)) for j in range(ret_heads)]
    return {"left": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": taps,
                     "scale": dim ** -0.5, "mask": {"size": window}, "rot": rot},
            "right": {"heads": ret_heads, "dim": ret_dim, "vdim": ret_vdim, "decay": decay,
                      "rot": {"dims": ret_dim, "base": 10000.0}},
            "left_scale": 0.8, "right_scale": 0.6}


def _ff(n):
    return {"kind": "dense", "ff": n}


def _moe(experts, top, ff, groups, keep, limit=7.0, scale=1.5):
    return {"kind": "moe", "router": {"experts": experts, "top": top, "scale": scale,
                                      "groups": {"count": groups, "keep": keep}},
            "expert": {"ff": ff, "limit": limit}}


def _preset(name, vocab, width, layers, bigram=(4093, 1009, 917)):
    return config_from_dict({"vocab": vocab, "width": width, "norm": {"eps": 1e-6},
                             "embedding": {"bigram": dict(zip(("buckets", "mul_prev", "mul_cur"), bigram))},
                             "layers": [{"type": PARALLEL if "left" in m else DELTA, "mixer": m, "mlp": f}
                                        for m, f in layers]}, name)


PRESETS = {
    # CPU-test sized
    "pitelorn-tiny": _preset("pitelorn-tiny", 320, 96, [
        (_par(4, 2, 16, 24, 20, 3, 3, 16, 8, rot_dims=8), _ff(128)),
        (_delta(4, 2, 16, 24, 4), _moe(6, 2, 40, 3, 2)),
        (_delta(3, 3, 12, 16, 2), None),
    ], bigram=(61, 7, 3)),
    # a 2048-wide stack (benchmarks): heads and dense layer of the sizes of nulazen-2k, as many active
    # expert weights per token as there (six of 32 experts for four and a shared one twice as wide)
    "pitelorn-2k": _preset("pitelorn-2k", 32768, 2048, [
        (_delta(16, 16, 128, 128, 4), _ff(8192)),
        (_par(16, 4, 128, 128, 1024, 4, 16, 128, 128), _moe(32, 6, 1024, 4, 2)),
        (_delta(16, 16, 128, 128, 4), _moe(32, 6, 1024, 4, 2)),
        (_par(16, 4, 128, 128, 1024, 4, 16, 128, 128), _moe(32, 6, 1024, 4, 2)),
    ]),
    # the same stack at 4096 width
    "pitelorn-4k": _preset("pitelorn-4k", 32768, 4096, [
        (_delta(32, 32, 128, 128, 4), _ff(14336)),
        (_par(32, 8, 128, 128, 2048, 4, 32, 128, 128), _moe(64, 8, 1408, 8, 4)),
        (_delta(32, 32, 128, 128, 4), _moe(64, 8, 1408, 8, 4)),
        (_par(32, 8, 128, 128, 2048, 4, 32, 128, 128), _moe(64, 8, 1408, 8, 4)),
    ]),
}


def _build(cfg, device, dtype, comm, max_model_len, quantization):
    return PitelornModel(cfg, device, dtype, comm, max_model_len, quantization)


register(Architecture(
    name="pitelorn",
    matches=lambda c: str(c.get("architecture", "")).lower() == "pitelorn",
    parse=lambda c, name: config_from_dict(c, name),
    build=_build,
    presets=PRESETS,
))
