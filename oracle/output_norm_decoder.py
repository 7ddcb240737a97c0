"""Plain, slow restatement of a decoder with norms on its sublayers' outputs (the Gulidra design), in numpy float64: differential
attention behind short convolutions, lightning attention (a linear attention with one decay per head), dense and routed feed-forwards.

One function per mechanism, written from the equations; nothing here is shared with the product path.  `Sequence` keeps what a
sequence carries from token to token, so that a prompt can also be fed in pieces.  Test infrastructure only.
"""
from __future__ import annotations

import json
import os

import numpy as np

from .latent_decoder import F, read_safetensors, rms_norm, sigmoid


def silu(z):
    return z * sigmoid(z)


def embedding(tokens, positions, table, scale, pos_table):
    return table[np.asarray(tokens)] * scale + pos_table[np.asarray(positions)]


def short_convolution(u, before, w):
    """u [tokens, channels] behind the taps - 1 values `before` ([taps - 1, channels], zeros at a sequence's start); w [channels, taps]:
    y_t = sum_j w[:, j] * u_(t - taps + 1 + j).  Returns (y, what the next portion needs)."""
    taps = w.shape[1]
    all_u = np.concatenate([before, u])
    y = np.zeros_like(u)
    for t in range(len(u)):
        for j in range(taps):
            y[t] += w[:, j] * all_u[t + j]
    return y, all_u[len(all_u) - (taps - 1):]


def unit_heads(x, n, dim, w, eps):
    """RMS norm over each of n groups of dim, one weight for all of them."""
    return rms_norm(x.reshape(-1, n, dim), w, eps)


def softmax_attend(q, k, v, scale, positions):
    """One map of one head: q [tokens, dim] at `positions`, k / v of positions 0 ..; causal."""
    s = (q @ k.T) * scale
    s[np.arange(len(k))[None, :] > np.asarray(positions)[:, None]] = -np.inf
    e = np.exp(s - s.max(axis=1, keepdims=True))
    return (e @ v) / e.sum(axis=1, keepdims=True)


def map_weight(lq1, lk1, lq2, lk2, diff):
    return np.exp(np.sum(lq1 * lk1)) - np.exp(np.sum(lq2 * lk2)) + diff


def join_maps(a1, a2, lam, diff, eps):
    o = a1 - lam * a2
    return o / np.sqrt(np.mean(o * o, axis=-1, keepdims=True) + eps) * (1.0 - diff)


def projected(h, T, name, state, taps):
    u = h @ T[name].T
    if not taps:
        return u
    before = state.get(name, np.zeros((taps - 1, u.shape[1]), dtype=F))
    y, state[name] = short_convolution(u, before, T[name + ".conv"])
    return y


def differential_keys(h, T, p, m, eps, state):
    """(keys [tokens, G, 2, dim] after convolution and norm, values [tokens, G, vdim] after convolution)."""
    G, taps = m["kv_heads"], m.get("conv") or 0
    k = unit_heads(projected(h, T, p + "k", state, taps), 2 * G, m["dim"], T[p + "k.norm"], eps)
    v = projected(h, T, p + "v", state, taps)
    return k.reshape(len(h), G, 2, m["dim"]), v.reshape(len(h), G, m["vdim"])


def differential_attention(h, keys, values, T, p, m, eps, state, positions):
    """Output before W_o of queries at `positions`; keys / values of positions 0 .. (these included)."""
    H, G, n = m["heads"], m["kv_heads"], len(h)
    q = unit_heads(projected(h, T, p + "q", state, m.get("conv") or 0), 2 * H, m["dim"], T[p + "q.norm"], eps).reshape(n, H, 2, m["dim"])
    lam = map_weight(T[p + "lq1"], T[p + "lk1"], T[p + "lq2"], T[p + "lk2"], m["diff"])
    gate = sigmoid(h @ T[p + "g"].T)
    out = np.zeros((n, H, m["vdim"]), dtype=F)
    for a in range(H):
        g = a // (H // G)
        maps = [softmax_attend(q[:, a, i], keys[:, g, i], values[:, g], m["scale"], positions) for i in (0, 1)]
        out[:, a] = join_maps(maps[0], maps[1], lam, m["diff"], eps) * gate[:, a:a + 1]
    return out.reshape(n, H * m["vdim"])


def lightning_recurrence(q, k, v, decay, S):
    """q, k [tokens, heads, dim], v [tokens, heads, vdim], S [heads, dim, vdim]: S <- decay_h S + k v^T, o = S^T q, token by token.
    Returns (o [tokens, heads, vdim], S)."""
    S = S.copy()
    o = np.zeros(v.shape, dtype=F)
    for t in range(len(q)):
        S = decay[:, None, None] * S + k[t][:, :, None] * v[t][:, None, :]
        o[t] = np.einsum("hdv,hd->hv", S, q[t])
    return o, S


def lightning_attention(h, T, p, m, eps, state):
    """Output before W_o."""
    n, H = len(h), m["heads"]
    q, k = (silu(h @ T[p + c].T).reshape(n, H, m["dim"]) for c in "qk")
    v = silu(h @ T[p + "v"].T).reshape(n, H, m["vdim"])
    S = state.get("S", np.zeros((H, m["dim"], m["vdim"]), dtype=F))
    o, state["S"] = lightning_recurrence(q, k, v, np.asarray(m["decay"], dtype=F), S)
    return rms_norm(o.reshape(n, H * m["vdim"]), T[p + "norm"], eps) * sigmoid(h @ T[p + "g"].T)


def gated_mlp(h, T, p):
    return (silu(h @ T[p + "gate"].T) * (h @ T[p + "up"].T)) @ T[p + "down"].T


def route(h, w_router, correction, top):
    """(chosen experts [tokens, top], their weights): softmax over all experts, the choice by score + correction, the weight the score."""
    z = h @ w_router.T
    e = np.exp(z - z.max(axis=1, keepdims=True))
    s = e / e.sum(axis=1, keepdims=True)
    chosen = np.argsort(-(s + correction), axis=1, kind="stable")[:, :top]
    return chosen, np.take_along_axis(s, chosen, axis=1)


def choice_margin(h, w_router, correction, top):
    """How far the choice is from another one, per token: the difference between the last chosen and the first left out, in units of their
    scores (how much a router logit would have to move); infinite where every expert is chosen."""
    z = h @ w_router.T
    e = np.exp(z - z.max(axis=1, keepdims=True))
    s = e / e.sum(axis=1, keepdims=True)
    if top >= s.shape[1]:
        return np.full(len(h), np.inf)
    c = s + correction
    order = np.argsort(-c, axis=1, kind="stable")
    pair = order[:, top - 1:top + 1]
    c2, s2 = np.take_along_axis(c, pair, axis=1), np.take_along_axis(s, pair, axis=1)
    return (c2[:, 0] - c2[:, 1]) / s2.max(axis=1)


def expert_mlp(h, T, p, r):
    """The last r.identity of the experts return their input."""
    chosen, weight = route(h, T[p + "router"], T[p + "correction"], r["top"])
    out = np.zeros_like(h)
    for e in range(r["experts"] + r.get("identity", 0)):
        t, j = np.nonzero(chosen == e)
        if len(t):
            y = h[t] if e >= r["experts"] else gated_mlp(h[t], T, f"{p}e{e}.")
            out[t] += weight[t, j][:, None] * y
    return out


# ---- the model ---------------------------------------------------------------------------------------------------------
class Model:
    def __init__(self, cfg: dict, tensors: dict):
        self.cfg = cfg
        self.T = {k: v.astype(F) for k, v in tensors.items()}
        self.eps = cfg["norm"]["eps"]

    @classmethod
    def load(cls, folder):
        with open(os.path.join(folder, "config.json")) as f:
            cfg = json.load(f)
        return cls(cfg, read_safetensors(os.path.join(folder, "model.safetensors")))

    def sequence(self):
        return Sequence(self)


class Sequence:
    def __init__(self, model):
        self.m, self.n = model, 0
        self.state = [dict() for _ in model.cfg["layers"]]
        self.kv = {}
        self.layer_outputs = []
        self.margins = []          # smallest choice_margin of every token fed so far

    def mixer(self, i, layer, x, pos):
        T, eps, m, p = self.m.T, self.m.eps, layer["mixer"], f"l{i}.mix."
        if layer["type"] == "lightning":
            y = lightning_attention(x, T, p, m, eps, self.state[i])
        else:
            src = m.get("kv_from")
            if src is None:
                new = differential_keys(x, T, p, m, eps, self.state[i])
                old = self.kv.get(i)
                self.kv[i] = new if old is None else tuple(np.concatenate([a, b]) for a, b in zip(old, new))
                src = i
            y = differential_attention(x, *self.kv[src], T, p, m, eps, self.state[i], pos)
        return y @ T[p + "o"].T

    def feed(self, tokens):
        """Logits [tokens, vocab] of the next tokens of the sequence."""
        cfg, T, eps = self.m.cfg, self.m.T, self.m.eps
        pos = np.arange(self.n, self.n + len(tokens))
        x = embedding(tokens, pos, T["embed"], cfg["embedding"]["scale"], T["pos"])
        mult = cfg["residual_mult"]
        self.layer_outputs = []
        margin = np.full(len(tokens), np.inf)
        for i, layer in enumerate(cfg["layers"]):
            p = f"l{i}."
            x = x + mult * rms_norm(self.mixer(i, layer, x, pos), T[p + "norm1"], eps)
            if layer.get("mlp"):
                l = layer["mlp"]
                if l["kind"] != "dense":
                    margin = np.minimum(margin, choice_margin(x, T[p + "mlp.router"], T[p + "mlp.correction"], l["router"]["top"]))
                y = gated_mlp(x, T, p + "mlp.") if l["kind"] == "dense" else expert_mlp(x, T, p + "mlp.", l["router"])
                x = x + mult * rms_norm(y, T[p + "norm2"], eps)
            self.layer_outputs.append(x)
        self.n += len(tokens)
        self.margins += margin.tolist()
        return rms_norm(x, T["final.norm"], eps) @ T["head"].T
