"""Small Fomunex configurations with random weights, written as model folders, for comparisons with oracle/prenorm_decoder.py."""
import copy

import numpy as np

from oracle import prenorm_decoder as pd
from pimosun_common import write_folder


def attention(heads, kv_heads, dim, vdim, window, cap, scale=None):
    return dict(type="attention", mixer=dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, mask=dict(size=window), softcap=cap,
                                             scale=scale if scale is not None else 2.0 * dim ** -0.5))


def mixing(heads, dim):
    return dict(type="wkv", mixer=dict(heads=heads, dim=dim))


def space(heads, groups, state, vdim, conv, norm_groups):
    return dict(type="mamba2", mixer=dict(heads=heads, groups=groups, state=state, vdim=vdim, conv=conv, norm_groups=norm_groups))


def dense(ff):
    return dict(kind="dense", ff=ff)


def experts(n, top, ff, limit):
    return dict(kind="moe", expert=dict(ff=ff, limit=limit), router=dict(experts=n, top=top))


def model(vocab, width, layers, eps=1e-5, positions=700, logit_scale=0.7, logit_softcap=12.0):
    """layers: (entry, feed-forward), or the number of the layer whose tensors are used."""
    out = []
    for l in layers:
        out.append(dict(l[0], mlp=l[1]) if isinstance(l, tuple) else l)
    for i, l in enumerate(out):
        if isinstance(l, int):
            j = l
            while isinstance(out[j], int):
                j = out[j]
            out[i] = dict(copy.deepcopy({k: v for k, v in out[j].items() if k != "weights_of"}), weights_of=l)
    return dict(architecture="Fomunex", vocab=vocab, width=width, norm=dict(eps=eps), max_positions=positions, logit_scale=logit_scale, logit_softcap=logit_softcap, layers=out)


def config_odd():
    """Sizes that fill no tile, windows that end inside pages, layers without feed-forward, tensors used by a later layer, by one after that, and by
    an earlier one."""
    return model(101, 84, [(space(6, 3, 20, 14, 4, 4), experts(6, 2, 24, 0.8)),
                           (mixing(5, 12), dense(50)),
                           (attention(6, 2, 20, 37, 45, 9.0), experts(9, 3, 40, 1.5)),
                           (attention(9, 3, 10, 12, 130, 30.0, scale=-0.9), None),
                           6,
                           0,
                           (mixing(2, 33), experts(5, 5, 17, 0.4)),
                           2,
                           4,
                           (space(5, 1, 33, 9, 2, 1), dense(17)),
                           (space(4, 4, 7, 21, 1, 12), None)], eps=1e-3)


def config_even():
    """Sizes that fill their tiles: the fast kernels' common case."""
    return model(320, 192, [(mixing(4, 64), dense(256)), (attention(8, 2, 64, 64, 96, 15.0), experts(16, 4, 128, 2.0)), (space(8, 2, 64, 32, 4, 8), dense(384)),
                            (attention(4, 2, 128, 64, 64, 25.0), experts(8, 2, 64, 1.1)), 0, 2], eps=1e-6, logit_scale=1.3, logit_softcap=20.0)


def config_wide():
    """Heads of the largest sizes served, others of real models' sizes."""
    return model(130, 160, [(attention(2, 1, 256, 256, 100, 20.0), None), (mixing(1, 256), experts(40, 6, 32, 1.0)), (space(3, 1, 256, 160, 4, 2), dense(96)),
                            (space(8, 2, 128, 64, 4, 2), None), (attention(3, 3, 160, 144, 70, 50.0), experts(4, 1, 32, 0.7)), (mixing(2, 128), None), 3], logit_scale=1.0, logit_softcap=30.0)


def config_one():
    """Everything that can be one is one."""
    return model(33, 32, [(attention(1, 1, 1, 1, 1, 1.0, scale=1.0), experts(1, 1, 1, 1.0)), (mixing(1, 1), dense(1)), (space(1, 1, 1, 1, 1, 1), None),
                          (attention(1, 1, 2, 1, 2, 1.0, scale=1.0), experts(2, 2, 3, 1.0)), 1], eps=0.1, logit_scale=1.0, logit_softcap=1.0)


CONFIGS = dict(odd=config_odd, even=config_even, wide=config_wide, one=config_one)


def random_config(seed):
    """Layers of any kind in any order, sizes of any kind."""
    rng = np.random.default_rng(seed)

    def one(*of):
        return of[int(rng.integers(len(of)))]
    layers = []
    for i in range(int(rng.integers(3, 8))):
        if i and rng.integers(5) == 0:
            layers.append(int(rng.integers(i)))
            continue
        kind = one("attention", "mixing", "space")
        sizes = (8, 12, 16, 24, 31, 32, 48, 64, 96, 100, 128)
        if kind == "attention":
            G, group = one(1, 2, 3, 4), one(1, 2, 4, 17)
            l = attention(G * group, G, one(*sizes), one(*sizes), one(1, 2, 17, 32, 63, 64, 65, 100, 128, 129, 400), one(2.0, 8.0, 30.0))
        elif kind == "mixing":
            l = mixing(int(rng.integers(1, 7)), one(*sizes))
        else:
            G, H, v = one(1, 2, 3), one(1, 2, 4), one(*sizes)
            l = space(G * H, G, one(*sizes), v, one(1, 2, 3, 4, 6), one(*[g for g in range(1, 9) if G * H * v % g == 0 and G * H * v // g > 3]))
        E = one(1, 2, 5, 12, 20)
        layers.append((l, one(None, dense(one(16, 40, 70, 129)), experts(E, int(rng.integers(1, min(4, E) + 1)), one(16, 40, 64), one(0.5, 1.0, 4.0)))))
    return model(one(64, 150, 257), one(48, 100, 128, 192), layers, eps=one(1e-5, 1e-4, 1e-3), positions=one(150, 1000), logit_scale=one(0.4, 1.0, 2.0), logit_softcap=one(5.0, 30.0))


def random_tensors(cfg, seed=0):
    rng = np.random.default_rng(seed)
    T, D = {}, cfg["width"]

    def mat(name, n, k, g=1.0):
        T[name] = (rng.standard_normal((n, k)) * g / np.sqrt(k)).astype(np.float32)

    def vec(name, n, mean=1.0, spread=0.2):
        T[name] = (mean + spread * rng.standard_normal(n)).astype(np.float32)
    T["embed"] = (3.0 * rng.standard_normal((cfg["vocab"], D))).astype(np.float32)
    T["pos"] = (1.0 * rng.standard_normal((cfg["max_positions"], D))).astype(np.float32)
    for i, l in enumerate(cfg["layers"]):
        if "weights_of" in l:
            continue
        p, m = f"l{i}.", l["mixer"]
        x = p + "mix."
        for q in "12" if l["mlp"] else "1":
            T[p + "norm" + q] = np.float32(rng.uniform(0.7, 1.4))
        if l["type"] == "attention":
            H, G = m["heads"], m["kv_heads"]
            for c, r in (("q", H * m["dim"]), ("k", G * m["dim"]), ("v", G * m["vdim"])):
                mat(x + c, r, D)
            vec(x + "sink", H, 1.0, 1.5)
            mat(x + "o", D, H * m["vdim"])
        elif l["type"] == "wkv":
            H, d = m["heads"], m["dim"]
            for c in "rkvgw":
                T[x + "mu." + c] = rng.uniform(-0.2, 1.2, size=D).astype(np.float32)
            for c in "rkvg":
                mat(x + c, H * d, D)
            rank = 3 + 9 * (i % 5)
            mat(x + "w1", rank, D)
            mat(x + "w2", H * d, rank)
            T[x + "w0"] = rng.uniform(-5.0, 1.0, size=H * d).astype(np.float32)
            T[x + "u"] = rng.standard_normal((H, d)).astype(np.float32)
            vec(x + "norm", H * d)
            mat(x + "o", D, H * d)
        else:
            H, inner = m["heads"], m["heads"] * m["vdim"]
            cols = inner + 2 * m["groups"] * m["state"]
            mat(x + "in", inner + cols + H, D)
            T[x + "conv"] = (rng.standard_normal((cols, m["conv"])) / np.sqrt(m["conv"]) * 1.5).astype(np.float32)
            vec(x + "conv.b", cols, 0.1, 0.4)
            T[x + "dt_bias"] = rng.uniform(-3.0, 0.5, size=H).astype(np.float32)
            T[x + "A_log"] = rng.uniform(-2.5, 1.5, size=H).astype(np.float32)
            vec(x + "D", H, 0.8, 0.5)
            vec(x + "norm", inner)
            mat(x + "o", D, inner)
        f = l["mlp"]
        if f and f["kind"] == "dense":
            mat(p + "mlp.up", f["ff"], D)
            mat(p + "mlp.down", D, f["ff"])
            T[p + "mlp.act"] = (np.array([0.8, -0.5, 0.3, 0.2]) + 0.2 * rng.standard_normal(4)).astype(np.float32)
        elif f:
            for e in range(f["router"]["experts"]):
                q = f"{p}mlp.e{e}."
                mat(q + "gate", f["expert"]["ff"], D, 1.5)
                mat(q + "up", f["expert"]["ff"], D, 1.5)
                mat(q + "down", D, f["expert"]["ff"], 0.1)         # another choice on a close call in bf16 moves little
            mat(p + "mlp.router", f["router"]["experts"], D, 3.0)
    T["final.norm"] = np.float32(1.2)
    mat("head", cfg["vocab"], D, 3.0)
    return T


def make_folder(path, name, seed=3):
    cfg = CONFIGS[name]()
    return write_folder(path, cfg, random_tensors(cfg, seed))


__all__ = ["CONFIGS", "pd", "random_config", "random_tensors", "make_folder", "write_folder", "model", "attention", "mixing", "space", "dense", "experts"]
