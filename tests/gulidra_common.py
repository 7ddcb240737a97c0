"""Small Gulidra configurations with random weights, written as model folders, for comparisons with oracle/output_norm_decoder.py."""
import numpy as np

from oracle import output_norm_decoder as od
from pimosun_common import write_folder


def attention(heads, kv_heads, dim, vdim, conv=3, diff=0.25, scale=None, kv_from=None):
    m = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale if scale is not None else 1.4 * dim ** -0.5, diff=diff)
    if conv:
        m["conv"] = conv
    if kv_from is not None:
        m["kv_from"] = kv_from
    return dict(type="attention", mixer=m)


def lightning(heads, dim, vdim, decay):
    return dict(type="lightning", mixer=dict(heads=heads, dim=dim, vdim=vdim, decay=[float(d) for d in decay]))


def dense(ff):
    return dict(kind="dense", ff=ff)


def experts(n, identity, top, ff):
    return dict(kind="moe", expert=dict(ff=ff), router=dict(experts=n, identity=identity, top=top))


def model(vocab, width, layers, eps=1e-5, scale=3.0, mult=0.8, positions=700):
    return dict(architecture="Gulidra", vocab=vocab, width=width, norm=dict(eps=eps), embedding=dict(scale=scale), residual_mult=mult, max_positions=positions,
                layers=[dict(l, mlp=m) for l, m in layers])


def config_odd():
    """Sizes that fill no tile, grouped heads, other taps in every layer, layers without feed-forward, readers of other layers' keys."""
    return model(101, 84, [(attention(6, 2, 20, 37, conv=4, diff=0.1), experts(7, 3, 3, 24)),
                           (lightning(3, 24, 40, [0.5, 0.93, 0.9995]), dense(56)),
                           (attention(3, 1, 40, 24, conv=2, diff=0.6), None),
                           (attention(4, 2, 20, 37, conv=5, diff=0.3, kv_from=0), experts(5, 0, 2, 33)),
                           (lightning(5, 9, 50, [0.2, 0.7, 0.9, 0.99, 1.0]), experts(3, 4, 5, 17)),
                           (attention(5, 1, 40, 24, conv=3, diff=0.2, kv_from=2), dense(40))], eps=2e-3, mult=0.6)


def config_even():
    """Sizes that fill their tiles: the fast kernels' common case."""
    return model(320, 256, [(attention(4, 4, 64, 128), experts(16, 2, 4, 128)), (lightning(4, 128, 128, [0.8, 0.95, 0.99, 0.999]), dense(512)),
                            (attention(8, 4, 64, 128, kv_from=0), dense(256))], eps=1e-6, scale=8.0, mult=1.0)


def config_wide():
    """Heads of the largest sizes served, more columns than one head's tiles."""
    return model(130, 160, [(attention(2, 1, 256, 256, conv=3), dense(96)), (attention(3, 3, 128, 128, conv=None, diff=0.8), None),
                            (lightning(2, 256, 160, [0.97, 0.999]), experts(40, 1, 6, 32)), (lightning(1, 256, 256, [0.99]), None)], scale=1.0)


def config_one():
    """Everything that can be one is one."""
    return model(33, 32, [(attention(1, 1, 1, 1, conv=1, diff=0.0, scale=1.0), experts(1, 0, 1, 1)), (lightning(1, 1, 1, [0.9]), dense(1)),
                          (lightning(1, 2, 3, [0.999]), experts(2, 1, 3, 5))], scale=1.0, mult=1.0, positions=200)


CONFIGS = dict(odd=config_odd, even=config_even, wide=config_wide, one=config_one)


def random_config(seed):
    """Layers of any kind in any order, sizes of any kind; readers of any earlier layer's keys.  The embedding outweighs what layers add, so
    that rounding where two maps nearly cancel stays small."""
    rng = np.random.default_rng(seed)

    def one(*of):
        return of[int(rng.integers(len(of)))]
    layers, own = [], []
    for i in range(int(rng.integers(2, 6))):
        kind = one("own", "own", "reader", "lightning")
        if kind == "lightning":
            H = int(rng.integers(1, 7))
            l = lightning(H, one(8, 16, 24, 32, 48, 64, 100), one(8, 16, 24, 32, 48, 72, 128), 1 - 2.0 ** -rng.uniform(0.5, 11, size=H))
        elif kind == "reader" and own:
            j = one(*own)
            m = layers[j][0]["mixer"]
            l = attention(m["kv_heads"] * one(1, 2, 3), m["kv_heads"], m["dim"], m["vdim"], one(1, 2, 3, 4), float(rng.uniform(0, 0.9)), kv_from=j)
        else:
            G = one(1, 2, 3, 4)
            l = attention(G * one(1, 2, 4, 17), G, one(8, 16, 24, 32, 48, 64, 96, 128), one(16, 32, 40, 64, 96, 128), one(None, 1, 2, 3, 4, 6), float(rng.uniform(0, 0.9)))
            own.append(i)
        E = one(2, 4, 6, 12, 24)
        layers.append((l, one(None, dense(one(30, 64, 200)), experts(E, one(0, 1, 3), int(rng.integers(1, min(E, 5) + 1)), one(16, 40, 64)))))
    return model(one(64, 150, 257), one(48, 100, 128, 192), layers, eps=one(1e-6, 1e-5, 1e-3), scale=one(4.0, 8.0, 15.0), mult=one(0.3, 0.7, 1.0), positions=150)


def random_tensors(cfg, seed=0):
    rng = np.random.default_rng(seed)
    T, D = {}, cfg["width"]

    def mat(name, n, k, g=1.0):
        T[name] = (rng.standard_normal((n, k)) * g / np.sqrt(k)).astype(np.float32)

    def vec(name, n, mean=1.0, spread=0.2):
        T[name] = (mean + spread * rng.standard_normal(n)).astype(np.float32)
    T["embed"] = rng.standard_normal((cfg["vocab"], D)).astype(np.float32)
    T["pos"] = (0.5 * rng.standard_normal((cfg["max_positions"], D))).astype(np.float32)
    for i, l in enumerate(cfg["layers"]):
        p, m = f"l{i}.", l["mixer"]
        x = p + "mix."
        vec(p + "norm1", D)
        H, dim, vdim = m["heads"], m["dim"], m["vdim"]
        if l["type"] == "lightning":
            for c, n in (("q", H * dim), ("k", H * dim), ("v", H * vdim), ("g", H * vdim)):
                mat(x + c, n, D, 1.5)
            vec(x + "norm", H * vdim)
        else:
            G = m["kv_heads"]
            for c, n in (("q", 2 * H * dim), ("k", 2 * G * dim), ("v", G * vdim)):
                if c != "q" and "kv_from" in m:
                    continue
                mat(x + c, n, D)
                if m.get("conv"):
                    T[x + c + ".conv"] = (rng.standard_normal((n, m["conv"])) / np.sqrt(m["conv"])).astype(np.float32)
                if c != "v":
                    vec(x + c + ".norm", dim, 1.2)
            for c in ("lq1", "lk1", "lq2", "lk2"):
                vec(x + c, dim, 0.0, 0.8 * dim ** -0.5)
            mat(x + "g", H, D)
        mat(x + "o", D, H * vdim)
        if l["mlp"]:
            vec(p + "norm2", D)
            def gated(q, ff):
                mat(q + "gate", ff, D)
                mat(q + "up", ff, D)
                mat(q + "down", D, ff)
            if l["mlp"]["kind"] == "dense":
                gated(p + "mlp.", l["mlp"]["ff"])
            else:
                r = l["mlp"]["router"]
                for e in range(r["experts"]):
                    gated(f"{p}mlp.e{e}.", l["mlp"]["expert"]["ff"])
                mat(p + "mlp.router", r["experts"] + r["identity"], D, 3.0)       # few experts carry the weight: a close call among the last moves little
                vec(p + "mlp.correction", r["experts"] + r["identity"], 0.0, 0.1)
    vec("final.norm", D)
    mat("head", cfg["vocab"], D)
    return T


def make_folder(path, name, seed=3):
    cfg = CONFIGS[name]()
    return write_folder(path, cfg, random_tensors(cfg, seed))


__all__ = ["CONFIGS", "od", "random_config", "random_tensors", "make_folder", "write_folder"]
