"""Logirax: a decoder-only model with norms before and after every sublayer
(x += norm1b(mixer(norm1 x)); x += norm2b(ff(norm2 x)), norm weights stored as offsets
from one) whose mixers read a token-shifted input: h + (h' - h) * shift with h = norm1 x
and h' the previous token's h, kept per layer in the sequence's state slot.

* Embedding: embed[token] * embedding.scale.
* Mixer ``attention``: grouped-query attention whose values are its keys as projected,
  with rotated and then normed q and k, capped scores mixed across the heads, a sliding
  window that also keeps the sequence's first tokens, and a sigmoid output gate
  (:class:`..models.mixers.TalkingHeadsAttention`).
* Mixer ``latent_attention``: latent attention with a latent for the queries too, rotary
  pairs of neighbours, a learned sink per head and a sigmoid gate per head
  (:class:`..models.mixers.LatentAttention`).
* Feed-forward (optional per layer): ``dense``, the clamped GLU
  (:class:`..models.mixers.GatedFF`), or ``moe``, silu-GLU experts chosen by their router
  logits and weighted by renormalised sigmoids, plus an ungated shared expert
  (:class:`..models.mixers.MoEFF`).
* Output: the model's norm, then the embedding table itself as the head, times
  ``logit_scale``.

Every size comes from ``config.json`` (keys: vocab, width, norm.eps, embedding.scale,
logit_scale, layers[].type / mixer / mlp; attention mixer{heads, kv_heads, dim, scale,
softcap, mask{size, keep_first}, rot{dims, base}}; latent mixer{heads, dim, rot_dim, vdim,
kv_rank, q_rank, scale, rot{base}}; mlp{kind, ff, limit} or {kind, router{experts, top,
scale}, expert{ff}, shared{ff}}) or from tensor shapes.  Tensor names: embed, final.norm,
l<i>.{norm1,norm1b,norm2,norm2b,shift}, l<i>.mix.{q,q.b,k,k.b,temp,talk,g,o,o.b} or
l<i>.mix.{dq,dq.norm,uq,dkv,dkv.norm,uk,uv,sink,g,o},
l<i>.mlp.{gate,up,down} or l<i>.mlp.{router,e<j>.*,shared.*}.

The model body (layer runs, residual, token shift, caches, logits) is
:class:`..models.stacked.StackedModel`.
"""
from __future__ import annotations

import dataclasses
import os
from typing import Dict, List, Optional, Tuple

import torch

from .mixers import GatedFF, LatentAttention, MoEFF, TalkingHeadsAttention
from .registry import Architecture, register
from .stacked import StackedLayer, StackedModel

ATTENTION, LATENT = "attention", "latent_attention"
DENSE, MOE = "dense", "moe"


@dataclasses.dataclass(frozen=True)
class LogiraxConfig:
    name: str
    vocab_size: int
    hidden_size: int
    rms_norm_eps: float
    embed_scale: float
    logit_scale: float
    layers: tuple                      # per layer: dict(type=, mixer=, mlp=)
    max_position_embeddings: int = 1 << 17
    bos_token_id: int = 0
    eos_token_ids: tuple = ()
    tie_word_embeddings: bool = True
    architecture = "logirax"

    @property
    def num_layers(self) -> int:
        return len(self.layers)

    def runs(self) -> List[Tuple[int, Optional[int]]]:
        return [(i, None) for i in range(len(self.layers))]

    def num_params(self) -> int:
        return sum(int(torch.Size(s).numel()) for s in tensor_shapes(self).values())

    def kv_bytes_per_token(self, dtype_bytes: int = 2) -> int:
        total = 0
        for l in self.layers:
            m = l["mixer"]
            total += (m["kv_rank"] + m["rot_dim"] if l["type"] == LATENT else 2 * m["kv_heads"] * m["dim"]) * dtype_bytes
        return total


def config_from_dict(c: dict, name: str = "logirax") -> LogiraxConfig:
    layers = []
    for i, l in enumerate(c["layers"]):
        m = dict(l["mixer"])
        if l["type"] == ATTENTION:
            m.setdefault("kv_heads", m["heads"])
            if m.setdefault("vdim", m["dim"]) != m["dim"]:
                raise ValueError(f"layer {i}: values are the keys as projected, so vdim must equal dim")
        elif l["type"] == LATENT:
            rot = m.get("rot") or {}
            if int(rot.get("dims", m["rot_dim"])) != m["rot_dim"]:
                raise ValueError(f"layer {i}: the whole rotated part is rotated, so rot.dims must equal rot_dim")
        else:
            raise ValueError(f"layer {i}: unknown mixer type {l['type']!r}")
        mlp = l.get("mlp")
        if mlp is not None:
            kind = mlp.get("kind", MOE if "router" in mlp else DENSE)
            if kind == DENSE:
                mlp = {"kind": DENSE, "ff": int(mlp["ff"]), "limit": float(mlp["limit"])}
            elif kind == MOE:
                mlp = {"kind": MOE, "router": dict(mlp["router"]), "expert": dict(mlp["expert"]),
                       "shared": dict(mlp["shared"]) if mlp.get("shared") else None}
            else:
                raise ValueError(f"layer {i}: unknown feed-forward kind {kind!r}")
        layers.append({"type": l["type"], "mixer": m, "mlp": mlp})
    return LogiraxConfig(name=name, vocab_size=int(c["vocab"]), hidden_size=int(c["width"]),
                         rms_norm_eps=float(c.get("norm", {}).get("eps", 1e-6)),
                         embed_scale=float((c.get("embedding") or {}).get("scale", 1.0)),
                         logit_scale=float(c.get("logit_scale", 1.0)), layers=tuple(layers),
                         max_position_embeddings=int(c.get("max_positions", 1 << 17)))


def config_to_dict(cfg: LogiraxConfig) -> dict:
    layers = []
    for l in cfg.layers:
        mlp = None
        if l["mlp"] is not None:
            mlp = {k: (dict(v) if isinstance(v, dict) else v) for k, v in l["mlp"].items() if v is not None}
        layers.append({"type": l["type"], "mixer": dict(l["mixer"]), "mlp": mlp})
    return {"architecture": "Logirax", "vocab": cfg.vocab_size, "width": cfg.hidden_size,
            "norm": {"eps": cfg.rms_norm_eps}, "embedding": {"scale": cfg.embed_scale},
            "logit_scale": cfg.logit_scale, "layers": layers}


def tensor_shapes(cfg: LogiraxConfig) -> Dict[str, tuple]:
    """Names and shapes of a checkpoint of this configuration (random init, tests)."""
    w, v = cfg.hidden_size, cfg.vocab_size
    t: Dict[str, tuple] = {"embed": (v, w), "final.norm": (w,)}
    for i, l in enumerate(cfg.layers):
        p, m, mlp = f"l{i}.", l["mixer"], l["mlp"]
        h, dk = m["heads"], m["dim"]
        t.update({p + "norm1": (w,), p + "norm1b": (w,), p + "shift": (w,)})
        q = p + "mix."
        if l["type"] == ATTENTION:
            g = m["kv_heads"]
            t.update({q + "q": (h * dk, w), q + "q.b": (h * dk,), q + "k": (g * dk, w), q + "k.b": (g * dk,),
                      q + "talk": (h, h), q + "temp": (h,), q + "g": (h * dk, w), q + "o": (w, h * dk), q + "o.b": (w,)})
        else:
            dr, dv, r, qr = m["rot_dim"], m["vdim"], m["kv_rank"], m["q_rank"]
            t.update({q + "dq": (qr, w), q + "dq.norm": (qr,), q + "uq": (h * (dk + dr), qr), q + "dkv": (r + dr, w),
                      q + "dkv.norm": (r,), q + "uk": (h * dk, r), q + "uv": (h * dv, r), q + "sink": (h,),
                      q + "g": (h, w), q + "o": (w, h * dv)})
        if mlp is None:
            continue
        t.update({p + "norm2": (w,), p + "norm2b": (w,)})
        glu = lambda at, ff: t.update({at + "gate": (ff, w), at + "up": (ff, w), at + "down": (w, ff)})   # noqa: E731
        if mlp["kind"] == DENSE:
            glu(p + "mlp.", mlp["ff"])
        else:
            for j in range(mlp["router"]["experts"]):
                glu(p + f"mlp.e{j}.", mlp["expert"]["ff"])
            t[p + "mlp.router"] = (mlp["router"]["experts"], w)
            if mlp["shared"]:
                glu(p + "mlp.shared.", mlp["shared"]["ff"])
    return t


def random_tensors(cfg: LogiraxConfig, seed: int = 0, dtype=torch.bfloat16, device="cpu") -> Dict[str, torch.Tensor]:
    """Random weights of the configuration's shapes: projections ~ N(0, 1/fan_in), offset
    norm weights near 0, plain norm weights near 1, shifts in (0, 1), head mixes near the
    identity, head factors near 1."""
    g = torch.Generator(device=device).manual_seed(seed)
    out: Dict[str, torch.Tensor] = {}
    for name, shape in tensor_shapes(cfg).items():
        leaf = name.split(".")[-1]
        r = torch.rand(shape, generator=g, device=device)
        n = torch.randn(shape, generator=g, device=device)
        if name == "embed":
            x = n
        elif leaf == "talk":
            x = torch.eye(shape[0], device=device) + 0.3 * n
        elif len(shape) == 2:
            x = n * shape[1] ** -0.5
        elif leaf == "temp":
            x = 1.0 + r
        elif leaf == "shift":
            x = r
        elif leaf == "sink":
            x = n
        elif leaf == "b":
            x = 0.2 * n
        elif name.endswith(("dq.norm", "dkv.norm")):     # plain norm weights
            x = 0.75 + 0.5 * r
        else:                                            # offsets from one
            x = 0.25 * (r - 0.5)
        out[name] = x.to(dtype)
    return out


def save_checkpoint(cfg: LogiraxConfig, tensors: Dict[str, torch.Tensor], out_dir: str):
    import json

    from safetensors.torch import save_file

    os.makedirs(out_dir, exist_ok=True)
    save_file({k: v.contiguous().cpu() for k, v in tensors.items()},
              os.path.join(out_dir, "model.safetensors"))
    with open(os.path.join(out_dir, "config.json"), "w") as f:
        json.dump(config_to_dict(cfg), f, indent=1)


class LogiraxModel(StackedModel):
    family = "Logirax"

    def load_tensors(self, get, has=lambda n: True):
        cfg, dev, dt = self.cfg, self.device, self.dtype
        eps, width = cfg.rms_norm_eps, cfg.hidden_size
        self.load_head(get, lambda n: n != "head" and has(n))     # the embedding table is the head
        self.embed_scale, self.logit_scale = cfg.embed_scale, cfg.logit_scale
        nw = lambda n: self.offset_norm_weight(get(n))   # noqa: E731
        self.final_norm = nw("final.norm")
        max_pos = max(self.max_model_len, 16) + 1
        self.layers = []
        for i, l in enumerate(cfg.layers):
            p, m, mlp = f"l{i}.", l["mixer"], l["mlp"]
            mix = lambda n, p=p: get(p + "mix." + n)   # noqa: E731
            rot = m.get("rot") or {}
            base = float(rot.get("base", 10000.0))
            if l["type"] == ATTENTION:
                mask = m.get("mask") or {}
                mixer = TalkingHeadsAttention(mix, width, m["heads"], m["kv_heads"], m["dim"],
                                              int(mask.get("size", 0)), int(mask.get("keep_first", 0)), m["scale"],
                                              m.get("softcap") or 0.0, int(rot.get("dims", 0)), base, eps, dt, dev,
                                              max_pos)
            else:
                mixer = LatentAttention(mix, width, m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"],
                                        m["scale"], m["rot_dim"], base, eps, dt, dev, max_pos, q_latent=True,
                                        interleaved=True, sink=True, head_gate=True)
            L = StackedLayer(l["type"], nw(p + "norm1"), nw(p + "norm1b"), mixer,
                             shift=get(p + "shift").to(dev, torch.float32).contiguous())
            if mlp is not None:
                L.norm2, L.norm2b = nw(p + "norm2"), nw(p + "norm2b")
                ff = lambda n, p=p: get(p + "mlp." + n)   # noqa: E731
                if mlp["kind"] == DENSE:
                    L.ff = GatedFF(ff, dt, dev, act="clamp_glu", limit=mlp["limit"])
                else:
                    r = mlp["router"]
                    L.ff = MoEFF(ff, r["experts"], r["top"], 0.0, 1, 1, None, dt, dev, routing="top_sigmoid",
                                 act="silu_glu", shared=bool(mlp["shared"]), shared_gate=False,
                                 route_scale=float(r.get("scale", 1.0)))
            self.layers.append(L)
        return self

    def random_tensors(self, seed: int, device):
        return random_tensors(self.cfg, seed, torch.bfloat16, device=device)


# ---------------------------------------------------------------------------------------
# registry: shapes for random-init runs (benchmarks, smoke tests)
# ---------------------------------------------------------------------------------------

def _att(heads, kv_heads, dim, window, keep, softcap=30.0, base=500000.0, rot_dims=None):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "scale": dim ** -0.5, "softcap": softcap,
            "mask": {"size": window, "keep_first": keep}, "rot": {"dims": rot_dims or dim, "base": base}}


def _lat(heads, dim, rot_dim, vdim, kv_rank, q_rank, base=500000.0):
    return {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "q_rank": q_rank,
            "scale": (dim + rot_dim) ** -0.5, "rot": {"dims": rot_dim, "base": base}}


def _moe(experts, top, ff, shared_ff, scale=1.5):
    return {"kind": MOE, "router": {"experts": experts, "top": top, "scale": scale}, "expert": {"ff": ff},
            "shared": {"ff": shared_ff} if shared_ff else None}


def _dense(ff, limit=7.0):
    return {"kind": DENSE, "ff": ff, "limit": limit}


def _preset(name, vocab, width, layers, scale=1.0):
    return config_from_dict({"vocab": vocab, "width": width, "norm": {"eps": 1e-6}, "embedding": {"scale": scale},
                             "logit_scale": 1.0,
                             "layers": [{"type": LATENT if "kv_rank" in m else ATTENTION, "mixer": m, "mlp": f}
                                        for m, f in layers]}, name)


PRESETS = {
    # CPU-test sized
    "logirax-tiny": _preset("logirax-tiny", 320, 80, [
        (_att(4, 2, 16, 20, 3, rot_dims=8), _dense(96)),
        (_lat(3, 16, 8, 12, 24, 20), _moe(6, 2, 32, 48)),
        (_att(4, 1, 16, 12, 2), None),
    ], scale=4.0),
    # a 2048-wide stack (benchmarks): three windowed layers per latent layer, sizes of heads,
    # latent, experts and dense layer as nulazen-2k's
    "logirax-2k": _preset("logirax-2k", 32768, 2048, [
        (_att(16, 4, 128, 1024, 64), _dense(8192)),
        (_att(16, 4, 128, 1024, 64), _moe(32, 4, 1024, 2048)),
        (_att(16, 4, 128, 1024, 64), _moe(32, 4, 1024, 2048)),
        (_lat(16, 128, 64, 128, 512, 1024), _moe(32, 4, 1024, 2048)),
    ], scale=16.0),
    # the same stack at 4096 width
    "logirax-4k": _preset("logirax-4k", 32768, 4096, [
        (_att(32, 8, 128, 2048, 64), _dense(14336)),
        (_att(32, 8, 128, 2048, 64), _moe(64, 6, 1408, 2816)),
        (_att(32, 8, 128, 2048, 64), _moe(64, 6, 1408, 2816)),
        (_lat(32, 128, 64, 128, 512, 1536), _moe(64, 6, 1408, 2816)),
    ], scale=16.0),
}


def _build(cfg, device, dtype, comm, max_model_len, quantization):
    return LogiraxModel(cfg, device, dtype, comm, max_model_len, quantization)


register(Architecture(
    name="logirax",
    matches=lambda c: str(c.get("architecture", "")).lower() == "logirax",
    parse=lambda c, name: config_from_dict(c, name),
    build=_build,
    presets=PRESETS,
))
