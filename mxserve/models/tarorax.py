"""Tarorax: a decoder whose config.json lists its layers and whose residual is `streams` vectors x_1 .. x_n per
token instead of one, all equal to the embedding at the start.  A sublayer (q = 1: the mixer, q = 2: the
feed-forward, when the layer has one) reads and writes them through learned coefficients:
    u = sum_s in_q[s] x_s,   y = ls_q * sublayer(norm_q(u)),   x_t <- sum_s mix_q[s, t] x_s + out_q[t] y
with RMS norms whose weights are stored as their difference from one and an element-wise layer scale ls_q.
The logits are embed times the final norm of sum_s x_s.

  gla            mixers.GatedLinearAttention: a decay per head and key channel from a low-rank pair
  attention      mixers.DifferentialAttention: two maps over the same values, the second subtracted; biases,
                 short convolutions, a query factor that grows with the position, bounded scores, no rotation
  mlp dense      feedforward.GatedFF with the tanh form of gelu
  mlp moe        feedforward.RoutedExperts: sigmoid scores with a correction for the choice, the best groups of
                 experts, renormalised and scaled weights on the outputs of ungated units with the exact gelu

The streams are fp32 from the embedding to the final norm, in one buffer [T, streams, width]: a sublayer's output
is biased, scaled and written into all of them, and the next sublayer's combination and norm taken, in one kernel
(seqmix.streams_update).  A layer's input projections are one GEMM, so are a dense feed-forward's gate and up.
One forward = one engine step over a flattened token batch: paged K/V through the block tables, fp32 recurrent and
convolution state in the runner's slots.
"""
from __future__ import annotations

import sys
from typing import Optional

import torch

from .. import ops
from ..ops import seqmix
from .config import ModelConfig
from .feedforward import FeedForward, GatedFF, RoutedExperts
from .hybrid import HybridLM, LayerPlan, plan_runs
from .mixers import DifferentialAttention, GatedLinearAttention, Mixer, StepContext


def build_mixer(kind: str, prefix: str, width: int, mc: dict) -> Mixer:
    if kind == "gla":
        return GatedLinearAttention(prefix, width, int(mc["heads"]), int(mc["dim"]), int(mc["vdim"]), float(mc["tau"]))
    if kind == "attention":
        return DifferentialAttention(prefix, width, int(mc["heads"]), int(mc.get("kv_heads", mc["heads"])), int(mc["dim"]),
                                     int(mc["vdim"]), float(mc["scale"]), float(mc["diff"]),
                                     float(mc.get("softcap") or 0.0), int(mc["conv"]), mc.get("q_temp"))
    raise ValueError(f"unknown mixer type {kind!r}")


def build_ff(prefix: str, width: int, mlp: Optional[dict]) -> Optional[FeedForward]:
    if not mlp:
        return None
    kind = mlp.get("kind", "dense")
    if kind == "dense":
        return GatedFF(prefix, width, int(mlp["ff"]), act="gelu_tanh")
    if kind == "moe":
        r = mlp["router"]
        g = r.get("groups") or {"count": 1, "keep": 1}
        return RoutedExperts(prefix, width, int(r["experts"]), int(r["top"]), int(mlp["expert"]["ff"]), None, renorm=True,
                             weigh="output", gated=False, act="gelu_erf", correction=True, groups=int(g["count"]),
                             keep=int(g["keep"]), scale=float(r.get("scale", 1.0)))
    raise ValueError(f"unknown feed-forward kind {kind!r}")


def mixers_of(ac: dict) -> list:
    return [build_mixer(l["type"], f"l{i}.mix.", int(ac["width"]), l["mixer"]) for i, l in enumerate(ac["layers"])]


def ffs_of(ac: dict) -> list:
    return [build_ff(f"l{i}.mlp.", int(ac["width"]), l.get("mlp")) for i, l in enumerate(ac["layers"])]


def layer_plan(ac: dict, block_size: int = 16, mixers: Optional[list] = None) -> LayerPlan:
    """Every layer runs once, in order, each over pages and a state of its own."""
    mixers = mixers or mixers_of(ac)
    return plan_runs([(i, None, False) for i in range(len(mixers))], mixers, block_size)


def weight_shapes(ac: dict, mixers: Optional[list] = None) -> dict:
    """Checkpoint tensor names and shapes."""
    W, V, n = int(ac["width"]), int(ac["vocab"]), int(ac["streams"])
    mixers = mixers or mixers_of(ac)
    ffs = ffs_of(ac)
    sh = {"embed": (V, W), "final.norm": (W,)}
    for i, m in enumerate(mixers):
        p = f"l{i}."
        for name, rows in m.proj_rows():
            sh[name] = (rows, W)
        sh.update(m.extra_shapes())
        if ffs[i] is not None:
            sh.update(ffs[i].shapes())
        for q in (1, 2) if ffs[i] is not None else (1,):
            sh[f"{p}norm{q}"] = sh[f"{p}ls{q}"] = (W,)
            sh[f"{p}hc{q}.in"] = sh[f"{p}hc{q}.out"] = (n,)
            sh[f"{p}hc{q}.mix"] = (n, n)
    return sh


def random_state(ac: dict, seed: int = 0, device="cpu") -> dict:
    """Random weights in checkpoint naming (fp32): projections ~ N(0, 1/fan_in); norms around their neutral
    value; layer scales around one half, the streams' matrices near the identity, their vectors near one;
    decays, corrections and routers spread so that each mechanism matters."""
    g = torch.Generator(device=device).manual_seed(seed)
    rnd = lambda shape: torch.randn(shape, generator=g, device=device)  # noqa: E731
    out = {}
    for name, shape in weight_shapes(ac).items():
        leaf = name.rsplit(".", 1)[-1]
        if leaf in ("norm1", "norm2") or name == "final.norm":
            t = 0.1 * rnd(shape)
        elif leaf == "norm":
            t = 1.0 + 0.1 * rnd(shape)
        elif leaf in ("ls1", "ls2"):
            t = 0.5 + 0.2 * rnd(shape)
        elif leaf == "mix" and len(shape) == 2 and ".hc" in name:
            t = torch.eye(shape[0], device=device) + 0.2 * rnd(shape)
        elif leaf == "in" and ".hc" in name:
            t = (1.0 + 0.5 * rnd(shape)) / shape[0]
        elif leaf == "out" and ".hc" in name:
            t = 1.0 + 0.5 * rnd(shape)
        elif name.endswith("a2.b"):
            t = 1.0 + 2.0 * rnd(shape)
        elif leaf == "b":
            t = 0.3 * rnd(shape)
        elif leaf in ("lq1", "lk1", "lq2", "lk2"):
            t = rnd(shape) * shape[0] ** -0.5
        elif leaf == "correction":
            t = 0.2 * rnd(shape)
        elif leaf == "router":
            t = 2.0 * rnd(shape) * shape[1] ** -0.5
        elif name == "embed":
            t = rnd(shape)
        else:
            t = rnd(shape) * shape[1] ** -0.5
        out[name] = t
    return out


class TaroraxLM(HybridLM):
    design = sys.modules[__name__]

    def __init__(self, cfg: ModelConfig, device, dtype: torch.dtype = torch.bfloat16, block_size: int = 16):
        super().__init__(cfg, device, dtype, block_size)
        self.streams = int(self.ac["streams"])
        self.ffs = ffs_of(self.ac)
        # the sublayers in execution order: (layer, 1 = mixer | 2 = feed-forward)
        self.subs = [(i, q) for i, f in enumerate(self.ffs) for q in ((1, 2) if f is not None else (1,))]

    def finish_weights(self, w: dict) -> None:
        for f in self.ffs:
            if f is not None:
                f.finish_weights(w)
        # what one update of the streams needs, in one fp32 vector: its mix and out, and the NEXT sublayer's
        # in (ones after the last: the sum of the streams)
        fp = {k: w.pop(k).to(torch.float32).reshape(-1) for k in [k for k in w if ".hc" in k]}
        ones = torch.ones(self.streams, dtype=torch.float32, device=w["embed"].device)
        ins = [fp[f"l{i}.hc{q}.in"] for i, q in self.subs] + [ones]
        w["_start.in"] = ins[0].contiguous()
        for k, (i, q) in enumerate(self.subs):
            w[f"l{i}.hc{q}"] = torch.cat([fp[f"l{i}.hc{q}.mix"], fp[f"l{i}.hc{q}.out"], ins[k + 1]]).contiguous()

    def lm_head_weight(self) -> torch.Tensor:
        return self.w["embed"]

    def forward(self, input_ids: torch.Tensor, md, kv_cache: torch.Tensor) -> torch.Tensor:
        """Final-normed hidden states of the rows md.logits_indices."""
        w, eps, dt = self.w, self.eps, self.dtype
        ctx = StepContext(md=md, cache=kv_cache, state=md.state, block_size=self.block_size, eps=eps)
        norms = [w[f"l{i}.norm{q}"] for i, q in self.subs] + [w["final.norm"]]
        X, h = seqmix.streams_start(input_ids, w["embed"], self.streams, w["_start.in"], norms[0], eps, 1.0, dt)
        tap = self.layer_tap
        for k, (i, q) in enumerate(self.subs):
            if q == 1:
                run, mx = self.plan.runs[i], self.mixers[i]
                y = mx.forward(self._split(ops.linear(h, w[f"l{i}.mix._in"]), mx), h, w, ctx, run.koff, run.voff, run.soff)
                bias = w[mx.out_bias] if mx.out_bias else None
            else:
                y, bias = self.ffs[i].forward(h, w), None
            h = seqmix.streams_update(X, y, w[f"l{i}.hc{q}"], eps, norms[k + 1], dt, bias=bias, scale=w[f"l{i}.ls{q}"],
                                      w_offset=1.0)
            if tap is not None and (k + 1 == len(self.subs) or self.subs[k + 1][1] == 1):
                tap.append(X.sum(1))
        return h.index_select(0, md.logits_indices)

    def compute_logits(self, hidden: torch.Tensor) -> torch.Tensor:
        """fp32 logits: the embedding table is the output projection."""
        return seqmix.softcap(ops.linear(hidden, self.w["embed"]), 0.0)
