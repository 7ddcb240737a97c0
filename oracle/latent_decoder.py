"""Plain, slow restatement of a parallel-block decoder with latent attention (the Pimosun design), in numpy float64.

One function per mechanism, written from the equations; nothing here is shared with the product path.  A sequence is
computed whole, token by token where that is simplest; `Sequence` keeps the same quantities between portions so that a
prompt can also be fed in pieces.  Test infrastructure only.
"""
from __future__ import annotations

import json
import math
import os
import struct

import numpy as np

F = np.float64


def bf16_to_f32(bits: np.ndarray) -> np.ndarray:
    return (bits.astype(np.uint32) << 16).view(np.float32)


def f32_to_bf16(x: np.ndarray) -> np.ndarray:
    """Round to nearest, ties to even."""
    u = np.ascontiguousarray(x, dtype=np.float32).view(np.uint32)
    return ((u + 0x7FFF + ((u >> 16) & 1)) >> 16).astype(np.uint16)


def read_safetensors(path: str) -> dict:
    """name -> float32 (bf16 / f32) or int32 array."""
    out = {}
    with open(path, "rb") as f:
        (n,) = struct.unpack("<Q", f.read(8))
        head = json.loads(f.read(n))
        body = f.read()
    for name, d in head.items():
        if name == "__metadata__":
            continue
        a, b = d["data_offsets"]
        raw = body[a:b]
        if d["dtype"] == "BF16":
            v = bf16_to_f32(np.frombuffer(raw, dtype="<u2"))
        elif d["dtype"] == "F32":
            v = np.frombuffer(raw, dtype="<f4")
        elif d["dtype"] == "I32":
            v = np.frombuffer(raw, dtype="<i4")
        else:
            raise ValueError(d["dtype"])
        out[name] = v.reshape(d["shape"])
    return out


def write_safetensors(path: str, tensors: dict) -> None:
    """name -> float array; written as bf16."""
    head, blobs, at = {}, [], 0
    for name, v in tensors.items():
        b = f32_to_bf16(np.asarray(v, dtype=np.float32)).astype("<u2").tobytes()
        head[name] = {"dtype": "BF16", "shape": list(np.shape(v)), "data_offsets": [at, at + len(b)]}
        blobs.append(b)
        at += len(b)
    h = json.dumps(head).encode()
    h += b" " * (-len(h) % 8)
    with open(path, "wb") as f:
        f.write(struct.pack("<Q", len(h)) + h + b"".join(blobs))


# ---- one function per mechanism -------------------------------------------------------------------------------------
def rms_norm(x, w, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps) * w


def layer_norm(x, w, eps):
    d = x - np.mean(x, axis=-1, keepdims=True)
    return d / np.sqrt(np.mean(d * d, axis=-1, keepdims=True) + eps) * w


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def bigram_row(prev, token, buckets, mul_prev, mul_cur):
    """Row of the pair table; prev None = the token opens its sequence."""
    if prev is None:
        return buckets
    return (int(prev) * int(mul_prev) + int(token) * int(mul_cur)) % int(buckets)


def rotation(rot):
    """(frequencies [dims / 2], factor on cos and sin)."""
    dims, base = rot["dims"], float(rot["base"])
    f = np.array([base ** (-2.0 * i / dims) for i in range(dims // 2)], dtype=F)
    sc = rot.get("scaling")
    if not sc:
        return f, 1.0

    def where(turns):
        return dims * math.log(sc["original"] / (2.0 * math.pi * turns)) / (2.0 * math.log(base))
    lo = max(math.floor(where(sc["fast"])), 0)
    hi = min(math.ceil(where(sc["slow"])), dims - 1)
    ramp = np.clip((np.arange(dims // 2) - lo) / max(hi - lo, 0.001), 0.0, 1.0)
    return f / sc["factor"] * ramp + f * (1.0 - ramp), 0.1 * math.log(sc["factor"]) + 1.0


def rotate(x, positions, rot):
    """x [tokens, ..., width]: its first rot.dims entries rotated pairwise (2 i, 2 i + 1)."""
    f, mag = rotation(rot)
    a = np.asarray(positions, dtype=F)[:, None] * f[None, :]
    cos, sin = np.cos(a) * mag, np.sin(a) * mag
    shape = [x.shape[0]] + [1] * (x.ndim - 2) + [len(f)]
    cos, sin = cos.reshape(shape), sin.reshape(shape)
    out = x.copy()
    n = rot["dims"]
    u, v = x[..., 0:n:2], x[..., 1:n:2]
    out[..., 0:n:2] = u * cos - v * sin
    out[..., 1:n:2] = v * cos + u * sin
    return out


def sink_softmax_attend(scores, values, sink):
    """scores [keys], values [keys, vdim], one sink logit: the sink takes part in the denominator only."""
    top = max(float(np.max(scores)), float(sink))
    e = np.exp(scores - top)
    return (e @ values) / (np.sum(e) + math.exp(float(sink) - top))


def latent_of(h, T, p, m, eps, positions):
    """What a layer keeps per token: (normed latent [tokens, kv_rank], rotated shared key part [tokens, rot_dim])."""
    both = h @ T[p + "dkv"].T
    c = rms_norm(both[:, :m["kv_rank"]], T[p + "dkv.norm"], eps)
    return c, rotate(both[:, m["kv_rank"]:], positions, m["rot"])


def latent_attention(h, latents, T, p, m, eps, positions):
    """h [tokens, width]; latents = (c, r) of the keys at positions 0 .. (all earlier and these); output before W_o."""
    H, dim, rd, vd = m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    n = h.shape[0]
    q = (rms_norm(h @ T[p + "dq"].T, T[p + "dq.norm"], eps) @ T[p + "uq"].T).reshape(n, H, dim + rd)
    qn, qr = q[:, :, :dim], rotate(q[:, :, dim:], positions, m["rot"])
    c, r = latents
    k = (c @ T[p + "uk"].T).reshape(-1, H, dim)
    v = (c @ T[p + "uv"].T).reshape(-1, H, vd)
    gate = sigmoid(h @ T[p + "g"].T)
    out = np.zeros((n, H, vd), dtype=F)
    for t in range(n):
        seen = int(positions[t]) + 1
        for a in range(H):
            s = (k[:seen, a] @ qn[t, a] + r[:seen] @ qr[t, a]) * m["scale"]
            out[t, a] = sink_softmax_attend(s, v[:seen, a], T[p + "sink"][a]) * gate[t, a]
    return out.reshape(n, H * vd)


def gated_mlp(h, T, p):
    return (gelu_tanh(h @ T[p + "gate"].T) * (h @ T[p + "up"].T)) @ T[p + "down"].T


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
    """One sequence's state: the token before, the number of tokens so far, the latents of the layers that make them."""

    def __init__(self, model):
        self.m, self.n, self.prev, self.lat = model, 0, None, {}
        self.layer_outputs = []

    def feed(self, tokens):
        """Logits [tokens, vocab] of the next tokens of the sequence."""
        cfg, T, eps = self.m.cfg, self.m.T, self.m.eps
        x = T["embed"][np.asarray(tokens)].copy()
        bg = cfg["embedding"].get("bigram") if cfg.get("embedding") else None
        if bg:
            for i, t in enumerate(tokens):
                x[i] += T["bigram"][bigram_row(self.prev if i == 0 else tokens[i - 1], t, bg["buckets"], bg["mul_prev"], bg["mul_cur"])]
        pos = np.arange(self.n, self.n + len(tokens))
        self.layer_outputs = []
        for i, layer in enumerate(cfg["layers"]):
            p, m = f"l{i}.", layer["mixer"]
            h = layer_norm(x, T[p + "norm1"], eps)
            src = m.get("kv_from", None)
            if src is None:
                new = latent_of(h, T, p + "mix.", m, eps, pos)
                old = self.lat.get(i)
                self.lat[i] = new if old is None else tuple(np.concatenate([a, b]) for a, b in zip(old, new))
                src = i
            y = latent_attention(h, self.lat[src], T, p + "mix.", m, eps, pos) @ T[p + "mix.o"].T
            if layer.get("mlp"):
                y = y + gated_mlp(h, T, p + "mlp.")
            x = x + y
            self.layer_outputs.append(x)
        self.n += len(tokens)
        self.prev = int(tokens[-1])
        return layer_norm(x, T["final.norm"], eps) @ T["head"].T
