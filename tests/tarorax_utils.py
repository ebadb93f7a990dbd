"""Helpers of the Tarorax tests: small configurations and checkpoints on disk.  The engine, replay and
error helpers are those of the Voletar tests (they know nothing of a design)."""
from __future__ import annotations

import json
import os

import torch

from mxserve.models.tarorax import random_state
from tests.voletar_utils import cut, engine, rel_err, replay  # noqa: F401


def diff_attention(heads=6, kv_heads=2, dim=24, vdim=40, scale=0.2, softcap=12.0, diff=0.35, conv=3, coef=0.25, every=16):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "softcap": softcap, "diff": diff,
            "conv": conv, "q_temp": {"coef": coef, "every": every}}


def gla(heads=3, dim=20, vdim=28, tau=8.0):
    return {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau}


def dense(ff=96):
    return {"kind": "dense", "ff": ff}


def moe(experts=12, top=3, ff=40, groups=4, keep=2, scale=1.5):
    return {"kind": "moe", "expert": {"ff": ff},
            "router": {"experts": experts, "top": top, "groups": {"count": groups, "keep": keep}, "scale": scale}}


def layer(mixer, mlp=None):
    return {"type": "gla" if "tau" in mixer else "attention", "mixer": mixer, "mlp": mlp}


def config(layers, width=112, vocab=320, streams=3, eps=1e-5):
    return {"architecture": "Tarorax", "width": width, "vocab": vocab, "streams": streams, "layers": layers, "norm": {"eps": eps}}


BASE = config([layer(gla(), moe()), layer(diff_attention(), dense()), layer(gla(heads=2, dim=36, vdim=16, tau=3.0)),
               layer(diff_attention(heads=4, kv_heads=4, dim=16, vdim=24, scale=0.3, softcap=25.0, diff=0.7, conv=5, coef=0.5, every=7),
                     moe(experts=6, top=2, ff=32, groups=2, keep=1, scale=0.8))])


def write_checkpoint(path, cfg: dict, seed: int = 0, tweak=None) -> dict:
    """config.json + model.safetensors (bf16) under `path`; returns the stored weights as float64 arrays."""
    from safetensors.torch import save_file
    os.makedirs(path, exist_ok=True)
    sd = {k: v.to(torch.bfloat16).contiguous() for k, v in random_state(cfg, seed).items()}
    if tweak:
        tweak(sd)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file(sd, os.path.join(path, "model.safetensors"))
    return {k: v.double().numpy() for k, v in sd.items()}
