"""A plain float64 implementation of the Tarorax design, one function or class per mechanism, one token
at a time.  It shares no code with mxserve: the tests compare the engine against it.

A model is (config dict, {tensor name: float64 numpy array}).  `Oracle.step(token)` feeds one token of
one sequence and returns (logits, the sum of the streams after every layer).
"""
from __future__ import annotations

import math

import numpy as np

_erf = np.vectorize(math.erf, otypes=[np.float64])


# ------------------------------------------------------------------------------------- small pieces
def unit_rms(x, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def offset_norm(x, w, eps):
    """RMS norm whose weight is stored as its difference from one."""
    return unit_rms(x, eps) * (1.0 + w)


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def gelu_erf(z):
    return 0.5 * z * (1.0 + _erf(z / math.sqrt(2.0)))


def conv_step(hist: list, u, w):
    """Output at the newest input u [channels] of the causal filter w [channels, taps]; `hist` holds the
    earlier inputs, newest last.  Inputs before the first are zero."""
    taps = w.shape[1]
    y = w[:, taps - 1] * u
    for back in range(1, taps):
        if back <= len(hist):
            y = y + w[:, taps - 1 - back] * hist[-back]
    return y


def query_temperature(pos: int, coef: float, every: float) -> float:
    return 1.0 + coef * math.log(math.floor((pos + 1) / every) + 1.0)


def capped_softmax_mix(scores, V, cap):
    """Scores bounded to (-cap, cap), softmax over all of them, weighted sum of the rows of V."""
    s = cap * np.tanh(scores / cap)
    e = np.exp(s - s.max())
    return (e @ V) / e.sum()


def layer_lambda(lq1, lk1, lq2, lk2, diff: float) -> float:
    return math.exp(float(lq1 @ lk1)) - math.exp(float(lq2 @ lk2)) + diff


# ------------------------------------------------------------------------------------- mixers
class DifferentialAttention:
    """Every head has two query maps over two key maps and one value; what the second map gathers is
    subtracted lambda times from what the first one gathers."""

    def __init__(self, mc: dict, w: dict, p: str, eps: float):
        self.H, self.G, self.dk, self.dv = int(mc["heads"]), int(mc["kv_heads"]), int(mc["dim"]), int(mc["vdim"])
        self.scale, self.cap, self.diff = float(mc["scale"]), float(mc["softcap"]), float(mc["diff"])
        self.coef, self.every = float(mc["q_temp"]["coef"]), float(mc["q_temp"]["every"])
        self.eps = eps
        self.w = {k[len(p):]: v for k, v in w.items() if k.startswith(p)}
        self.past = {"q": [], "k": [], "v": []}  # projected values before the filter
        self.keys, self.vals = [], []

    def _project(self, name, h):
        u = self.w[name] @ h + self.w[name + ".b"]
        y = conv_step(self.past[name], u, self.w[name + ".conv"])
        self.past[name].append(u)
        return y

    def step(self, h, pos):
        w, H, G = self.w, self.H, self.G
        q = self._project("q", h).reshape(H, 2, self.dk) * query_temperature(pos, self.coef, self.every)
        self.keys.append(self._project("k", h).reshape(G, 2, self.dk))
        self.vals.append(self._project("v", h).reshape(G, self.dv))
        K, V = np.stack(self.keys), np.stack(self.vals)  # [n, G, 2, dk], [n, G, dv]
        lam = layer_lambda(w["lq1"], w["lk1"], w["lq2"], w["lk2"], self.diff)
        out = np.empty((H, self.dv))
        for hd in range(H):
            g = hd // (H // G)
            a = [capped_softmax_mix((K[:, g, m] @ q[hd, m]) * self.scale, V[:, g], self.cap) for m in (0, 1)]
            out[hd] = unit_rms(a[0] - lam * a[1], self.eps) * (1.0 - self.diff)
        return w["o"] @ (out.reshape(-1) * sigmoid(w["g"] @ h)) + w["o.b"]


class GatedLinearAttention:
    """S <- diag(alpha) S + k v^T, o = S^T q, with one decay per head and key channel."""

    def __init__(self, mc: dict, w: dict, p: str, eps: float):
        self.H, self.dk, self.dv, self.tau = int(mc["heads"]), int(mc["dim"]), int(mc["vdim"]), float(mc["tau"])
        self.eps = eps
        self.w = {k[len(p):]: v for k, v in w.items() if k.startswith(p)}
        self.S = np.zeros((self.H, self.dk, self.dv))

    def step(self, h, pos):
        w, H = self.w, self.H
        q = (w["q"] @ h).reshape(H, self.dk) / math.sqrt(self.dk)
        k = (w["k"] @ h).reshape(H, self.dk)
        v = (w["v"] @ h).reshape(H, self.dv)
        alpha = (sigmoid(w["a2"] @ (w["a1"] @ h) + w["a2.b"]) ** (1.0 / self.tau)).reshape(H, self.dk)
        o = np.empty((H, self.dv))
        for hd in range(H):
            self.S[hd] = alpha[hd][:, None] * self.S[hd] + np.outer(k[hd], v[hd])
            o[hd] = self.S[hd].T @ q[hd]
        o = unit_rms(o, self.eps) * w["norm"]
        return w["o"] @ (o.reshape(-1) * silu(w["g"] @ h))


# ------------------------------------------------------------------------------------- feed-forward
def dense_ff(h, w, p):
    return w[p + "down"] @ (gelu_tanh(w[p + "gate"] @ h) * (w[p + "up"] @ h))


def choose_experts(z, correction, router: dict):
    """Router logits z [E] -> (chosen experts, their weights, how far the nearest other choice was)."""
    E, top = int(router["experts"]), int(router["top"])
    n, keep = int(router["groups"]["count"]), int(router["groups"]["keep"])
    s = sigmoid(z)
    c = s + correction
    per = c.reshape(n, E // n)
    gs = np.sort(per, axis=1)[:, ::-1][:, :2].sum(axis=1)
    gorder = np.argsort(-gs, kind="stable")
    margin = float(gs[gorder[keep - 1]] - gs[gorder[keep]]) if keep < n else math.inf
    open_ = np.full((n, E // n), -np.inf)
    for g in gorder[:keep]:
        open_[g] = per[g]
    c = open_.reshape(-1)
    order = np.argsort(-c, kind="stable")
    chosen = order[:top]
    if top < E:
        margin = min(margin, float(c[order[top - 1]] - c[order[top]]))
    wt = s[chosen]
    return chosen, wt / (wt.sum() + 1e-20) * float(router["scale"]), margin


def routed_ff(h, w, p, mlp):
    chosen, wt, margin = choose_experts(w[p + "router"] @ h, w[p + "correction"], mlp["router"])
    y = np.zeros_like(h)
    for e, a in zip(chosen, wt):
        y = y + a * (w[f"{p}e{int(e)}.down"] @ gelu_erf(w[f"{p}e{int(e)}.up"] @ h))
    return y, margin


# ------------------------------------------------------------------------------------- the streams
def streams_in(X, w_in):
    """X [streams, width] -> what a sublayer reads."""
    return w_in @ X


def streams_out(X, mix, w_out, y):
    """Stream t becomes sum over s of mix[s, t] times stream s, plus w_out[t] y."""
    return mix.T @ X + np.outer(w_out, y)


# ------------------------------------------------------------------------------------- the model
class Oracle:
    def __init__(self, cfg: dict, w: dict):
        self.cfg, self.w = cfg, {k: np.asarray(v, dtype=np.float64) for k, v in w.items()}
        self.eps, self.n = float(cfg["norm"]["eps"]), int(cfg["streams"])
        kinds = {"gla": GatedLinearAttention, "attention": DifferentialAttention}
        self.mixers = [kinds[l["type"]](l["mixer"], self.w, f"l{i}.mix.", self.eps) for i, l in enumerate(cfg["layers"])]
        self.pos = 0
        self.margins = []  # per token: the smallest gap between a chosen and a left-out expert or group

    def step(self, token: int):
        w, eps = self.w, self.eps
        X = np.tile(w["embed"][token], (self.n, 1))
        sums, margin = [], math.inf
        for i, l in enumerate(self.cfg["layers"]):
            p = f"l{i}."
            y = self.mixers[i].step(offset_norm(streams_in(X, w[p + "hc1.in"]), w[p + "norm1"], eps), self.pos)
            X = streams_out(X, w[p + "hc1.mix"], w[p + "hc1.out"], y * w[p + "ls1"])
            mlp = l.get("mlp")
            if mlp:
                h = offset_norm(streams_in(X, w[p + "hc2.in"]), w[p + "norm2"], eps)
                if mlp.get("kind", "dense") == "dense":
                    y = dense_ff(h, w, p + "mlp.")
                else:
                    y, m = routed_ff(h, w, p + "mlp.", mlp)
                    margin = min(margin, m)
                X = streams_out(X, w[p + "hc2.mix"], w[p + "hc2.out"], y * w[p + "ls2"])
            sums.append(X.sum(0))
        self.pos += 1
        self.margins.append(margin)
        return w["embed"] @ offset_norm(X.sum(0), w["final.norm"], eps), sums


def run(cfg: dict, w: dict, tokens, margins=None) -> tuple:
    """(logits [n, vocab], stream sums [layers, n, width]) of one sequence; a list passed as `margins`
    receives every token's routing margin."""
    o = Oracle(cfg, w)
    lg, st = [], []
    for t in tokens:
        a, b = o.step(int(t))
        lg.append(a)
        st.append(b)
    if margins is not None:
        margins.extend(o.margins)
    return np.stack(lg), np.stack([np.stack(s) for s in st]).transpose(1, 0, 2)
