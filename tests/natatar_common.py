"""Small Natatar configurations with random weights, written as model folders, for comparisons with oracle/stream_decoder.py."""
import numpy as np

from oracle import stream_decoder as sd
from pimosun_common import write_folder


def attention(heads, kv_heads, dim, vdim, v_mix=None, scale=None):
    m = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale if scale is not None else 1.3 * dim ** -0.5)
    if v_mix is not None:
        m["v_mix"] = v_mix
    return dict(type="attention", mixer=m)


def parallel(left, right, rot_dims=None, base=300.0, scaling=None, cap=9.0, scales=(0.7, 1.2), scale=None):
    """left: heads, kv_heads, dim, vdim; right: heads, dim, vdim."""
    H, G, dim, vdim = left
    rot = dict(base=base, dims=rot_dims if rot_dims is not None else dim // 2 * 2)
    if scaling:
        rot["scaling"] = scaling
    l = dict(heads=H, kv_heads=G, dim=dim, vdim=vdim, scale=scale if scale is not None else 1.1 * dim ** -0.5, rot=rot)
    return dict(type="parallel", mixer=dict(left=l, left_scale=scales[0], right=dict(heads=right[0], dim=right[1], vdim=right[2], gate_cap=cap), right_scale=scales[1]))


def delta(heads, kv_heads, dim, vdim, conv):
    return dict(type="channel_delta", mixer=dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, conv=conv))


def experts(n, top, ff, groups=None, scale=None):
    r = dict(experts=n, top=top)
    if groups:
        r["groups"] = dict(count=groups[0], keep=groups[1])
    if scale is not None:
        r["scale"] = scale
    return dict(kind="moe", expert=dict(ff=ff), router=r)


def model(vocab, width, streams, layers, eps=1e-5, scale=3.0, mult=0.5):
    return dict(architecture="Natatar", vocab=vocab, width=width, streams=streams, norm=dict(eps=eps), embedding=dict(scale=scale), residual_mult=mult,
                layers=[dict(l, mlp=m) for l, m in layers])


YARN = dict(factor=6.0, original=64, fast=8.0, slow=0.5)


def config_odd():
    """Sizes that fill no tile, values mixed across other layers and not at all, part of a head rotated, other taps, layers without feed-forward; an eps
    that lets the normalizer of the matrix memory show through the norm behind it."""
    return model(101, 84, 3, [(attention(6, 2, 20, 37, v_mix=False), experts(6, 2, 24, (3, 2), 1.7)),
                              (delta(6, 3, 20, 37, 4), None),
                              (parallel((3, 1, 21, 24), (5, 19, 30), rot_dims=10, scaling=YARN), experts(9, 3, 40, (3, 2))),
                              (attention(4, 2, 24, 18, v_mix=True), experts(5, 5, 33, None, 0.5)),
                              (attention(9, 3, 10, 12, v_mix=True, scale=-0.4), None),
                              (delta(2, 1, 33, 50, 2), experts(8, 3, 17, (2, 1), 2.0)),
                              (parallel((4, 4, 12, 20), (2, 40, 9), cap=3.0, scales=(1.5, -0.4)), None),
                              (attention(2, 1, 30, 36, v_mix=True), experts(4, 2, 24, (4, 3)))], eps=0.1, mult=0.4)


def config_even():
    """Sizes that fill their tiles: the fast kernels' common case."""
    return model(320, 256, 4, [(parallel((4, 2, 64, 128), (4, 64, 64), scaling=dict(factor=4.0, original=128, fast=16.0, slow=1.0)), experts(16, 4, 128, (4, 2), 2.5)),
                               (attention(8, 2, 64, 64, v_mix=True), experts(8, 2, 128, (4, 3))), (delta(4, 2, 128, 128, 4), experts(8, 2, 64)),
                               (attention(4, 2, 128, 64, v_mix=True), experts(8, 4, 64, (2, 1)))], eps=1e-6, scale=8.0, mult=0.7)


def config_wide():
    """Heads of the largest sizes served, more streams than one launch form's."""
    return model(130, 160, 5, [(parallel((2, 1, 256, 256), (2, 256, 160), rot_dims=64), None), (attention(3, 3, 160, 144), experts(40, 6, 32, (10, 3), 1.3)),
                               (delta(2, 2, 256, 256, 3), None), (parallel((2, 2, 128, 96), (1, 130, 256), scales=(0.9, 0.8)), experts(4, 1, 32)),
                               (delta(3, 1, 192, 96, 3), None)], scale=1.0, mult=0.8)


def config_one():
    """Everything that can be one is one."""
    return model(33, 32, 1, [(attention(1, 1, 1, 1, v_mix=True, scale=1.0), experts(1, 1, 1, (1, 1))), (parallel((1, 1, 2, 1), (1, 1, 1), scales=(1.0, 1.0), scale=1.0), None),
                             (delta(1, 1, 1, 1, 1), experts(2, 1, 5, (2, 1))), (attention(1, 1, 3, 1, v_mix=True, scale=1.0), experts(2, 2, 3))], scale=1.0, mult=1.0)


CONFIGS = dict(odd=config_odd, even=config_even, wide=config_wide, one=config_one)


def random_config(seed):
    """Layers of any kind in any order, sizes of any kind."""
    rng = np.random.default_rng(seed)

    def one(*of):
        return of[int(rng.integers(len(of)))]
    layers = []
    v_cols = one(16, 24, 36, 64, 96)                # value columns of the layers that mix values
    for _ in range(int(rng.integers(2, 7))):
        kind = one("attention", "parallel", "delta")
        G, group = one(1, 2, 3, 4), one(1, 2, 4, 17)
        sizes = (8, 12, 16, 24, 31, 32, 48, 64, 96, 100, 128)
        if kind == "attention":
            mixed = bool(rng.integers(3))
            G = one(*[g for g in (1, 2, 3, 4) if v_cols % g == 0]) if mixed else G
            l = attention(G * group, G, one(*sizes), v_cols // G if mixed else one(*sizes), v_mix=mixed)
        elif kind == "parallel":
            dim = one(*sizes)
            l = parallel((G * group, G, dim, one(*sizes)), (int(rng.integers(1, 7)), one(*sizes), one(*sizes)), rot_dims=int(rng.integers(1, dim // 2 + 1)) * 2,
                         base=one(50.0, 1e4), scaling=one(None, YARN, dict(factor=2.0, original=4096, fast=32.0, slow=1.0)), cap=one(2.0, 8.0, 15.0),
                         scales=(float(rng.uniform(0.3, 1.3)), float(rng.uniform(0.3, 1.3))))
        else:
            l = delta(G * one(1, 2, 3), G, one(*sizes), one(*sizes), one(1, 2, 3, 4, 6))
        groups = one(None, (1, 1), (2, 1), (2, 2), (4, 3), (5, 2))
        count, keep = groups or (1, 1)
        E = count * one(1, 2, 3, 6)
        layers.append((l, one(None, experts(E, int(rng.integers(1, min(5, keep * E // count) + 1)), one(16, 40, 64), groups, one(None, 0.7, 2.0)))))
    return model(one(64, 150, 257), one(48, 100, 128, 192), one(1, 2, 3, 4, 6), layers, eps=one(1e-6, 1e-5, 1e-3), scale=one(4.0, 8.0, 15.0), mult=one(0.2, 0.5, 1.0))


def random_tensors(cfg, seed=0):
    rng = np.random.default_rng(seed)
    T, D, s = {}, cfg["width"], cfg["streams"]

    def mat(name, n, k, g=1.0):
        T[name] = (rng.standard_normal((n, k)) * g / np.sqrt(k)).astype(np.float32)

    def vec(name, n, mean=1.0, spread=0.2):
        T[name] = (mean + spread * rng.standard_normal(n)).astype(np.float32)
    T["embed"] = rng.standard_normal((cfg["vocab"], D)).astype(np.float32)
    for i, l in enumerate(cfg["layers"]):
        p, m = f"l{i}.", l["mixer"]
        x = p + "mix."
        for q in "12" if l["mlp"] else "1":
            vec(p + "norm" + q, D, 0.0, 0.3)
            vec(f"{p}hc{q}.in", s, 1.0 / s, 0.3)
            vec(f"{p}hc{q}.out", s, 1.0, 0.3)
            T[f"{p}hc{q}.mix"] = (np.eye(s) * 0.8 + 0.2 / s + 0.15 * rng.standard_normal((s, s))).astype(np.float32)

        def heads(y, n, biases, norms):
            G = n["kv_heads"]
            for c, r in (("q", n["heads"] * n["dim"]), ("k", G * n["dim"]), ("v", G * n["vdim"])):
                mat(y + c, r, D)
                if biases:
                    vec(y + c + ".b", r, 0.0, 0.5)
                if norms and c != "v":
                    vec(y + c + ".norm", r, 1.2)
            mat(y + "o", D, n["heads"] * n["vdim"])
        if l["type"] == "attention":
            heads(x, m, True, True)
            T[x + "vmix"] = np.float32(0.4 + 0.1 * i)
        elif l["type"] == "parallel":
            heads(x + "left.", m["left"], False, False)
            mat(x + "left.g", m["left"]["heads"] * m["left"]["vdim"], D)
            n, y = m["right"], x + "right."
            H, v = n["heads"], n["heads"] * n["vdim"]
            for c, r in (("q", H * n["dim"]), ("k", H * n["dim"]), ("v", v), ("g", v), ("i", H), ("f", H)):
                mat(y + c, r, D, 2.0 if c in "if" else 1.0)
            mat(y + "o", D, v)
            vec(y + "norm", v)
            vec(y + "i.b", H, 0.0, 1.5)
            vec(y + "f.b", H, 3.0, 2.0)
        else:
            H, G = m["heads"], m["kv_heads"]
            for c, r in (("q", G * m["dim"]), ("k", G * m["dim"]), ("v", H * m["vdim"])):
                mat(x + c, r, D)
                T[x + c + ".conv"] = (rng.standard_normal((r, m["conv"])) / np.sqrt(m["conv"])).astype(np.float32)
            mat(x + "b", H, D, 2.0)
            T[x + "A_log"] = rng.uniform(-2.0, 1.5, size=H).astype(np.float32)
            vec(x + "dt_bias", H * m["dim"], -2.5, 1.5)
            vec(x + "norm", m["vdim"])
            ra, rg = 3 + 5 * (i % 4), 40 - 7 * (i % 3)
            mat(x + "a1", ra, D)
            mat(x + "a2", H * m["dim"], ra)
            mat(x + "g1", rg, D)
            mat(x + "g2", H * m["vdim"], rg)
            mat(x + "o", D, H * m["vdim"])
        if l["mlp"]:
            r, ff = l["mlp"]["router"], l["mlp"]["expert"]["ff"]
            for e in range(r["experts"]):
                q = f"{p}mlp.e{e}."
                mat(q + "gate", ff, D)
                mat(q + "up", ff, D)
                mat(q + "down", D, ff)
            mat(p + "mlp.router", r["experts"], D, 3.0)       # few experts carry the weight: a close call among the last moves little
    vec("final.norm", D, 0.0, 0.3)
    return T


def make_folder(path, name, seed=3):
    cfg = CONFIGS[name]()
    return write_folder(path, cfg, random_tensors(cfg, seed))


__all__ = ["CONFIGS", "sd", "random_config", "random_tensors", "make_folder", "write_folder"]
