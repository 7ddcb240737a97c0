"""Plain, slow restatement of a decoder whose residual is several mixed streams (the Natatar design), in numpy float64: attention with
normed projections and values shared along the depth, attention beside a matrix memory, a delta rule with one decay per key channel,
experts chosen within the best groups.

One function per mechanism, written from the equations; nothing here is shared with the product path.  `Sequence` keeps what a
sequence carries from token to token, so that a prompt can also be fed in pieces.  Test infrastructure only.
"""
from __future__ import annotations

import json
import os

import numpy as np

from .latent_decoder import F, read_safetensors, rms_norm, rotate, sigmoid
from .output_norm_decoder import gated_mlp, short_convolution, silu, softmax_attend


def around_zero_norm(x, w, eps):
    """RMS norm whose weight is stored less one."""
    return rms_norm(x, 1.0 + w, eps)


def log_sigmoid(z):
    return -np.logaddexp(0.0, -z)


def softplus(z):
    return np.logaddexp(0.0, z)


# ---- streams --------------------------------------------------------------------------------------------------------------
def read_streams(X, w_in):
    """X [streams, tokens, width]: what a sublayer reads, before its norm."""
    return np.tensordot(w_in, X, axes=(0, 0))


def write_streams(X, mix, w_out, y, mult):
    """Every stream from all old ones, mix[from, to], and its share of the sublayer's output."""
    return np.stack([sum(mix[s, t] * X[s] for s in range(len(X))) + mult * w_out[t] * y for t in range(len(X))])


# ---- attention ------------------------------------------------------------------------------------------------------------
def mix_values(v, first, lam):
    return (1.0 - lam) * v + lam * first


def attend_heads(q, k, v, scale, positions):
    """q [tokens, heads, dim] at `positions`, k [keys, kv_heads, dim], v [keys, kv_heads, vdim] of positions 0 ..; concatenated heads."""
    n, H, G = len(q), q.shape[1], k.shape[1]
    return np.concatenate([softmax_attend(q[:, a], k[:, a // (H // G)], v[:, a // (H // G)], scale, positions) for a in range(H)], axis=1).reshape(n, -1)


def kept(state, **new):
    """Keys and values of all tokens so far."""
    for c, x in new.items():
        state[c] = np.concatenate([state[c], x]) if c in state else x
    return [state[c] for c in new]


def normed_attention(h, T, p, m, eps, state, positions, first):
    """(output before W_o, this layer's own values): biases, norms over whole projections, no positions; `first` None = values stay as they are."""
    n, H, G = len(h), m["heads"], m["kv_heads"]
    q, k, v = (h @ T[p + c].T + T[p + c + ".b"] for c in "qkv")
    q, k = rms_norm(q, T[p + "q.norm"], eps), rms_norm(k, T[p + "k.norm"], eps)
    own = v
    if first is not None:
        v = mix_values(v, first, T[p + "vmix"])
    k, v = kept(state, k=k.reshape(n, G, -1), v=v.reshape(n, G, -1))
    return attend_heads(q.reshape(n, H, -1), k, v, m["scale"], positions), own


def gated_attention(h, T, p, m, state, positions):
    """Output before W_o: rotated queries and keys, a gate per column."""
    n, H, G = len(h), m["heads"], m["kv_heads"]
    q, k, v = ((h @ T[p + c].T).reshape(n, r, -1) for c, r in (("q", H), ("k", G), ("v", G)))
    k, v = kept(state, k=rotate(k, positions, m["rot"]), v=v)
    return attend_heads(rotate(q, positions, m["rot"]), k, v, m["scale"], positions) * sigmoid(h @ T[p + "g"].T)


# ---- matrix memory ----------------------------------------------------------------------------------------------------------
def soft_cap(z, cap):
    return cap * np.tanh(z / cap)


def memory_recurrence(q, k, v, i, f, S, n, m):
    """q, k [tokens, heads, dim], v [tokens, heads, vdim], log gates i, f [tokens, heads]; S [heads, dim, vdim], n [heads, dim], m [heads]."""
    o = np.zeros(v.shape, dtype=F)
    for t in range(len(q)):
        top = np.maximum(f[t] + m, i[t])
        keep, add = np.exp(f[t] + m - top), np.exp(i[t] - top)
        S = keep[:, None, None] * S + add[:, None, None] * k[t][:, :, None] * v[t][:, None, :]
        n = keep[:, None] * n + add[:, None] * k[t]
        m = top
        below = np.maximum(np.abs(np.sum(n * q[t], axis=1)), np.exp(-m)) + 1e-6
        o[t] = np.einsum("hdv,hd->hv", S, q[t]) / below[:, None]
    return o, S, n, m


def head_norm(o, eps):
    return o / np.sqrt(np.mean(o * o, axis=-1, keepdims=True) + eps)


def matrix_memory(h, T, p, m, eps, state):
    """Output before W_o."""
    N, H, d, e = len(h), m["heads"], m["dim"], m["vdim"]
    q, k = ((h @ T[p + c].T).reshape(N, H, d) for c in "qk")
    v = (h @ T[p + "v"].T).reshape(N, H, e)
    i = soft_cap(h @ T[p + "i"].T + T[p + "i.b"], m["gate_cap"])
    f = log_sigmoid(soft_cap(h @ T[p + "f"].T + T[p + "f.b"], m["gate_cap"]))
    S, n, top = state.get("S", np.zeros((H, d, e))), state.get("n", np.zeros((H, d))), state.get("m", np.zeros(H))
    o, state["S"], state["n"], state["m"] = memory_recurrence(q * d ** -0.5, k, v, i, f, S, n, top)
    return head_norm(o, eps).reshape(N, H * e) * T[p + "norm"] * sigmoid(h @ T[p + "g"].T)


# ---- delta rule -------------------------------------------------------------------------------------------------------------
def convolved(h, T, name, state):
    u, w = h @ T[name].T, T[name + ".conv"]
    before = state.get(name, np.zeros((w.shape[1] - 1, u.shape[1]), dtype=F))
    y, state[name] = short_convolution(u, before, w)
    return silu(y)


def unit(x):
    return x / np.sqrt(np.sum(x * x, axis=-1, keepdims=True) + 1e-6)


def channel_decay(a, A_log, dt_bias):
    """a [tokens, heads, dim], one A_log a head, dt_bias [heads, dim]."""
    return np.exp(-np.exp(A_log)[:, None] * softplus(a + dt_bias))


def delta_recurrence(q, k, v, g, beta, S):
    """q, k, g [tokens, heads, dim], v [tokens, heads, vdim], beta [tokens, heads], S [heads, dim, vdim]."""
    o = np.zeros(v.shape, dtype=F)
    for t in range(len(q)):
        S = g[t][:, :, None] * S
        u = beta[t][:, None] * (v[t] - np.einsum("hdv,hd->hv", S, k[t]))
        S = S + k[t][:, :, None] * u[:, None, :]
        o[t] = np.einsum("hdv,hd->hv", S, q[t])
    return o, S


def channel_delta(h, T, p, m, eps, state):
    """Output before W_o."""
    N, H, G, d, e = len(h), m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k = (unit(convolved(h, T, p + c, state).reshape(N, G, d)) for c in "qk")
    v = convolved(h, T, p + "v", state).reshape(N, H, e)
    share = np.arange(H) // (H // G)
    g = channel_decay((h @ T[p + "a1"].T @ T[p + "a2"].T).reshape(N, H, d), T[p + "A_log"], T[p + "dt_bias"].reshape(H, d))
    o, state["S"] = delta_recurrence(q[:, share] * d ** -0.5, k[:, share], v, g, sigmoid(h @ T[p + "b"].T), state.get("S", np.zeros((H, d, e))))
    return (head_norm(o, eps) * T[p + "norm"]).reshape(N, H * e) * sigmoid(h @ T[p + "g1"].T @ T[p + "g2"].T)


# ---- experts ----------------------------------------------------------------------------------------------------------------
def expert_scores(h, w_router):
    z = h @ w_router.T
    e = np.exp(z - z.max(axis=1, keepdims=True))
    return e / e.sum(axis=1, keepdims=True)


def allowed_experts(s, count, keep):
    """Which experts lie in the `keep` groups whose best score is largest."""
    best = s.reshape(len(s), count, -1).max(axis=2)
    order = np.argsort(-best, axis=1, kind="stable")[:, :keep]
    ok = np.zeros(best.shape, dtype=bool)
    np.put_along_axis(ok, order, True, axis=1)
    return np.repeat(ok, s.shape[1] // count, axis=1)


def route(h, w_router, r):
    """(chosen experts [tokens, top], their weights)."""
    s = expert_scores(h, w_router)
    g = r.get("groups") or dict(count=1, keep=1)
    c = np.where(allowed_experts(s, g["count"], g["keep"]), s, -np.inf)
    chosen = np.argsort(-c, axis=1, kind="stable")[:, :r["top"]]
    return chosen, np.take_along_axis(s, chosen, axis=1) * r.get("scale", 1.0)


def choice_margin(h, w_router, r):
    """How far the choice is from another one, per token: how much router logits would have to differ less, for the last chosen group against
    the next and the last chosen expert against the next; infinite where nothing is left out."""
    s = expert_scores(h, w_router)
    g = r.get("groups") or dict(count=1, keep=1)
    z = np.log(s)
    out = np.full(len(h), np.inf)
    best = np.sort(z.reshape(len(h), g["count"], -1).max(axis=2), axis=1)[:, ::-1]
    if g["keep"] < g["count"]:
        out = best[:, g["keep"] - 1] - best[:, g["keep"]]
    c = np.sort(np.where(allowed_experts(s, g["count"], g["keep"]), z, -np.inf), axis=1)[:, ::-1]
    if r["top"] < c.shape[1]:
        out = np.minimum(out, c[:, r["top"] - 1] - c[:, r["top"]])
    return out


def expert_mlp(h, T, p, r):
    chosen, weight = route(h, T[p + "router"], r)
    out = np.zeros_like(h)
    for e in range(r["experts"]):
        t, j = np.nonzero(chosen == e)
        if len(t):
            out[t] += weight[t, j][:, None] * gated_mlp(h[t], T, f"{p}e{e}.")
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
        self.state = [dict(left={}, right={}) for _ in model.cfg["layers"]]
        self.layer_outputs = []
        self.margins = []          # smallest choice_margin of every token fed so far

    def mixer(self, i, layer, h, pos, first):
        """(output, the layer's own values where later layers may take them)."""
        T, eps, m, p, st = self.m.T, self.m.eps, layer["mixer"], f"l{i}.mix.", self.state[i]
        if layer["type"] == "attention":
            y, own = normed_attention(h, T, p, m, eps, st, pos, first if m.get("v_mix") else None)
            return y @ T[p + "o"].T, own if m.get("v_mix") else None
        if layer["type"] == "parallel":
            left = gated_attention(h, T, p + "left.", m["left"], st["left"], pos) @ T[p + "left.o"].T
            right = matrix_memory(h, T, p + "right.", m["right"], eps, st["right"]) @ T[p + "right.o"].T
            return m["left_scale"] * left + m["right_scale"] * right, None
        assert layer["type"] == "channel_delta"
        return channel_delta(h, T, p, m, eps, st) @ T[p + "o"].T, None

    def feed(self, tokens):
        """Logits [tokens, vocab] of the next tokens of the sequence."""
        cfg, T, eps = self.m.cfg, self.m.T, self.m.eps
        pos = np.arange(self.n, self.n + len(tokens))
        X = np.stack([T["embed"][np.asarray(tokens)] * cfg["embedding"]["scale"]] * cfg["streams"])
        mult, first = cfg.get("residual_mult", 1.0), None
        self.layer_outputs = []
        margin = np.full(len(tokens), np.inf)
        for i, layer in enumerate(cfg["layers"]):
            p = f"l{i}."

            def sublayer(X, q, f):
                hc = f"{p}hc{q}."
                y = f(around_zero_norm(read_streams(X, T[hc + "in"]), T[f"{p}norm{q}"], eps))
                return write_streams(X, T[hc + "mix"], T[hc + "out"], y, mult)

            def mix(h):
                nonlocal first
                y, own = self.mixer(i, layer, h, pos, first)
                if first is None:
                    first = own
                return y

            def feed_forward(h):
                nonlocal margin
                margin = np.minimum(margin, choice_margin(h, T[p + "mlp.router"], layer["mlp"]["router"]))
                return expert_mlp(h, T, p + "mlp.", layer["mlp"]["router"])
            X = sublayer(X, 1, mix)
            if layer.get("mlp"):
                X = sublayer(X, 2, feed_forward)
            self.layer_outputs.append(X.sum(axis=0))
        self.n += len(tokens)
        self.margins += margin.tolist()
        return around_zero_norm(X.sum(axis=0), T["final.norm"], eps) @ T["embed"].T
