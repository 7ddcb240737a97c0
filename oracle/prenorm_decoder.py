"""Plain, slow restatement of a pre-norm decoder (the Fomunex design), in numpy float64: attention within a window whose scores are capped
and fall off with distance, with a sink in the denominator; a recurrence over mixes of neighbouring tokens with one decay per key channel
(RWKV-style); a state space recurrence with one decay a head behind a short convolution (Mamba-2); feed-forwards with a normed polynomial
as activation and experts whose weight scales their input.

One function per mechanism, written from the equations; nothing here is shared with the product path.  `Sequence` keeps what a
sequence carries from token to token, so that a prompt can also be fed in pieces.  Test infrastructure only.
"""
from __future__ import annotations

import json
import os

import numpy as np

from .latent_decoder import F, read_safetensors, sigmoid
from .output_norm_decoder import short_convolution, silu


def root_norm(x, eps):
    """x over its root mean square along the last axis."""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def scalar_norm(x, g, eps):
    """RMS norm whose weight is a scalar."""
    return root_norm(x, eps) * g


def soft_cap(z, cap):
    return z if cap is None else cap * np.tanh(z / cap)


def softplus(z):
    return np.logaddexp(0.0, z)


def embedding(tokens, positions, table, pos_table):
    return table[np.asarray(tokens)] + pos_table[np.asarray(positions)]


# ---- attention ------------------------------------------------------------------------------------------------------------
def slope(head, heads):
    return 2.0 ** (-8.0 * (head + 1) / heads)


def seen(i, j, window):
    """Whether position i sees position j."""
    return (j <= i) & (i - j < window) if window is not None else j <= i


def attend_head(q, k, v, positions, scale, cap, falloff, window, sink):
    """One head: q [tokens, dim] at `positions`, k / v of positions 0 .. ."""
    i, j = np.asarray(positions)[:, None], np.arange(len(k))[None, :]
    s = soft_cap((q @ k.T) * scale, cap) - falloff * (i - j)
    s = np.where(seen(i, j, window), s, -np.inf)
    top = np.maximum(s.max(axis=1, keepdims=True), sink)
    e = np.exp(s - top)
    return (e @ v) / (e.sum(axis=1, keepdims=True) + np.exp(sink - top))


def windowed_attention(h, T, p, m, eps, state, positions):
    """Output before W_o."""
    n, H, G = len(h), m["heads"], m["kv_heads"]
    q, k, v = ((h @ T[p + c].T).reshape(n, r, -1) for c, r in (("q", H), ("k", G), ("v", G)))
    q, k = root_norm(q, eps), root_norm(k, eps)
    for c, x in (("k", k), ("v", v)):
        state[c] = np.concatenate([state[c], x]) if c in state else x
    window = (m.get("mask") or {}).get("size")
    out = [attend_head(q[:, a], state["k"][:, a // (H // G)], state["v"][:, a // (H // G)], positions, m["scale"], m.get("softcap"), slope(a, H), window, T[p + "sink"][a])
           for a in range(H)]
    return np.concatenate(out, axis=1)


# ---- time mixing ------------------------------------------------------------------------------------------------------------
def shifted(h, before):
    """The token before each: `before` for the first."""
    return np.concatenate([before[None, :], h[:-1]])


def token_mix(h, h_before, mu):
    return h + (h_before - h) * mu


def channel_decay(z):
    return np.exp(-np.exp(z))


def bonus_recurrence(r, k, v, w, u, S):
    """r, k, w [tokens, heads, dim], v [tokens, heads, vdim], u [heads, dim], S [heads, dim, vdim]."""
    o = np.zeros(v.shape, dtype=F)
    for t in range(len(r)):
        kv = k[t][:, :, None] * v[t][:, None, :]
        o[t] = np.einsum("hdv,hd->hv", S + u[:, :, None] * kv, r[t])
        S = w[t][:, :, None] * S + kv
    return o, S


def time_mixing(h, T, p, m, eps, state):
    """Output before W_o."""
    n, H, d = len(h), m["heads"], m["dim"]
    before = shifted(h, state.get("h", np.zeros(h.shape[1], dtype=F)))
    state["h"] = h[-1]
    mix = {c: token_mix(h, before, T[p + "mu." + c]) for c in "rkvgw"}
    r, k, v = ((mix[c] @ T[p + c].T).reshape(n, H, d) for c in "rkv")
    w = channel_decay(np.tanh(mix["w"] @ T[p + "w1"].T) @ T[p + "w2"].T + T[p + "w0"]).reshape(n, H, d)
    o, state["S"] = bonus_recurrence(r, k, v, w, T[p + "u"], state.get("S", np.zeros((H, d, d), dtype=F)))
    return root_norm(o, eps).reshape(n, H * d) * T[p + "norm"] * silu(mix["g"] @ T[p + "g"].T)


# ---- state space ------------------------------------------------------------------------------------------------------------
def scalar_decay(dt, A_log):
    return np.exp(-np.exp(A_log) * dt)


def space_recurrence(x, B, C, dt, decay, D, S):
    """x [tokens, heads, vdim], B, C [tokens, heads, state], dt, decay [tokens, heads], D [heads], S [heads, state, vdim]."""
    y = np.zeros(x.shape, dtype=F)
    for t in range(len(x)):
        S = decay[t][:, None, None] * S + dt[t][:, None, None] * B[t][:, :, None] * x[t][:, None, :]
        y[t] = np.einsum("hnv,hn->hv", S, C[t]) + D[:, None] * x[t]
    return y, S


def gated_group_norm(y, z, groups, w, eps):
    """The gate first, then each of `groups` equal parts over its own root mean square."""
    y = y * silu(z)
    return root_norm(y.reshape(len(y), groups, -1), eps).reshape(y.shape) * w


def state_space(h, T, p, m, eps, state):
    """Output before W_o."""
    n, H, e, N, G = len(h), m["heads"], m["vdim"], m["state"], m["groups"]
    inner = H * e
    z, xBC, dt = np.split(h @ T[p + "in"].T, [inner, 2 * inner + 2 * G * N], axis=1)
    w = T[p + "conv"]
    y, state["conv"] = short_convolution(xBC, state.get("conv", np.zeros((w.shape[1] - 1, xBC.shape[1]), dtype=F)), w)
    x, B, C = np.split(silu(y + T[p + "conv.b"]), [inner, inner + G * N], axis=1)
    group = np.arange(H) // (H // G)
    dt = softplus(dt + T[p + "dt_bias"])
    y, state["S"] = space_recurrence(x.reshape(n, H, e), B.reshape(n, G, N)[:, group], C.reshape(n, G, N)[:, group], dt, scalar_decay(dt, T[p + "A_log"]), T[p + "D"],
                                     state.get("S", np.zeros((H, N, e), dtype=F)))
    return gated_group_norm(y.reshape(n, inner), z, m["norm_groups"], T[p + "norm"], eps)


# ---- feed-forwards ----------------------------------------------------------------------------------------------------------
def poly_norm(z, a, eps):
    return a[0] * root_norm(z, eps) + a[1] * root_norm(z ** 2, eps) + a[2] * root_norm(z ** 3, eps) + a[3]


def poly_mlp(h, T, p, eps):
    return poly_norm(h @ T[p + "up"].T, T[p + "act"], eps) @ T[p + "down"].T


def limited_gate(g, u, limit):
    g, u = np.minimum(g, limit), np.clip(u, -limit, limit)
    return g * sigmoid(1.702 * g) * (u + 1.0)


def expert(h, T, p, limit):
    return limited_gate(h @ T[p + "gate"].T, h @ T[p + "up"].T, limit) @ T[p + "down"].T


def route(h, w_router, top):
    """(chosen experts [tokens, top], their scores)."""
    s = sigmoid(h @ w_router.T)
    chosen = np.argsort(-s, axis=1, kind="stable")[:, :top]
    return chosen, np.take_along_axis(s, chosen, axis=1)


def choice_margin(h, w_router, top):
    """By how much the last chosen expert's router logit is above the first left out, per token; infinite where every expert is chosen."""
    z = np.sort(h @ w_router.T, axis=1)[:, ::-1]
    return z[:, top - 1] - z[:, top] if top < z.shape[1] else np.full(len(h), np.inf)


def routed_mlp(h, T, p, m):
    chosen, weight = route(h, T[p + "router"], m["router"]["top"])
    out = np.zeros_like(h)
    for e in range(m["router"]["experts"]):
        t, j = np.nonzero(chosen == e)
        if len(t):
            out[t] += expert(weight[t, j][:, None] * h[t], T, f"{p}e{e}.", m["expert"]["limit"])
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


def tensors_of(layers, i):
    """The layer whose tensors layer i uses."""
    while layers[i].get("weights_of") is not None:
        i = layers[i]["weights_of"]
    return i


class Sequence:
    def __init__(self, model):
        self.m, self.n = model, 0
        self.state = [dict() for _ in model.cfg["layers"]]
        self.layer_outputs = []
        self.margins = []          # smallest choice_margin of every token fed so far

    def feed(self, tokens):
        """Logits [tokens, vocab] of the next tokens of the sequence."""
        cfg, T, eps = self.m.cfg, self.m.T, self.m.eps
        pos = np.arange(self.n, self.n + len(tokens))
        x = embedding(tokens, pos, T["embed"], T["pos"])
        self.layer_outputs = []
        margin = np.full(len(tokens), np.inf)
        for i, layer in enumerate(cfg["layers"]):
            p, m, st = f"l{tensors_of(cfg['layers'], i)}.", layer["mixer"], self.state[i]
            h = scalar_norm(x, T[p + "norm1"], eps)
            if layer["type"] == "attention":
                y = windowed_attention(h, T, p + "mix.", m, eps, st, pos)
            elif layer["type"] == "wkv":
                y = time_mixing(h, T, p + "mix.", m, eps, st)
            else:
                assert layer["type"] == "mamba2"
                y = state_space(h, T, p + "mix.", m, eps, st)
            x = x + y @ T[p + "mix.o"].T
            if layer.get("mlp"):
                h = scalar_norm(x, T[p + "norm2"], eps)
                if layer["mlp"]["kind"] == "dense":
                    x = x + poly_mlp(h, T, p + "mlp.", eps)
                else:
                    margin = np.minimum(margin, choice_margin(h, T[p + "mlp.router"], layer["mlp"]["router"]["top"]))
                    x = x + routed_mlp(h, T, p + "mlp.", layer["mlp"])
            self.layer_outputs.append(x)
        self.n += len(tokens)
        self.margins += margin.tolist()
        logits = scalar_norm(x, T["final.norm"], eps) @ T["head"].T * cfg.get("logit_scale", 1.0)
        return soft_cap(logits, cfg.get("logit_softcap"))
