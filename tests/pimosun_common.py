"""Small Pimosun configurations with random weights, written as model folders, and comparisons with oracle/latent_decoder.py."""
import importlib
import json
import os

import numpy as np

from oracle import latent_decoder as ld

m40 = importlib.import_module("m40-llm_amd")
layered = importlib.import_module("m40-llm_amd.layered")


def mixer(heads, dim, rot_dim, vdim, kv_rank, q_rank, base=10000.0, scaling=None, scale=None, kv_from=None):
    m = dict(heads=heads, dim=dim, rot_dim=rot_dim, vdim=vdim, kv_rank=kv_rank, q_rank=q_rank,
             scale=scale if scale is not None else 1.3 * (dim + rot_dim) ** -0.5, rot=dict(base=base, dims=rot_dim))
    if scaling:
        m["rot"]["scaling"] = scaling
    if kv_from is not None:
        m["kv_from"] = kv_from
    return m


def layer(m, ff):
    return dict(type="latent_attention", mixer=m, mlp=None if ff is None else dict(kind="dense", ff=ff))


YARN = dict(factor=6.0, original=64, fast=8.0, slow=0.5)


def config_odd():
    """Sizes that fill no tile, layers that differ, a layer without feed-forward, a reader of another layer's entries."""
    return dict(architecture="Pimosun", vocab=101, width=80, norm=dict(eps=3e-3),
                embedding=dict(bigram=dict(buckets=37, mul_prev=11, mul_cur=5)),
                layers=[layer(mixer(3, 24, 8, 20, 40, 36, 500.0, YARN), 56),
                        layer(mixer(5, 10, 12, 7, 56, 20, 100.0), None),
                        layer(mixer(5, 18, 8, 33, 40, 50, 500.0, YARN, kv_from=0), 72),
                        layer(mixer(2, 16, 12, 24, 56, 33, 100.0, kv_from=1), 40)])


def config_even():
    """Sizes that fill their tiles; no pair table, no rotation scaling."""
    return dict(architecture="Pimosun", vocab=320, width=256, norm=dict(eps=1e-6), embedding={},
                layers=[layer(mixer(4, 64, 32, 64, 256, 128), 512), layer(mixer(4, 64, 32, 64, 256, 128, kv_from=0), 512)])


def config_wide():
    """The head sizes of a large model on a narrow stream."""
    return dict(architecture="Pimosun", vocab=200, width=128, norm=dict(eps=1e-5),
                embedding=dict(bigram=dict(buckets=1, mul_prev=0, mul_cur=1)),
                layers=[layer(mixer(9, 128, 64, 128, 512, 96, 10000.0, dict(factor=1.0, original=4096, fast=32.0, slow=1.0)), 160)])


def config_one():
    """Everything that can be one is one."""
    return dict(architecture="Pimosun", vocab=33, width=32, norm=dict(eps=1e-5),
                embedding=dict(bigram=dict(buckets=7, mul_prev=1, mul_cur=1)),
                layers=[layer(mixer(1, 1, 2, 1, 1, 1, 50.0, dict(factor=2.0, original=4, fast=2.0, slow=1.0), scale=1.0), 1)])


CONFIGS = dict(odd=config_odd, even=config_even, wide=config_wide, one=config_one)


def random_tensors(cfg, seed=0, gain=1.6):
    rng = np.random.default_rng(seed)
    T = {}

    def mat(name, n, k, g=1.0):
        T[name] = (rng.standard_normal((n, k)) * g / np.sqrt(k)).astype(np.float32)

    def vec(name, n, mean=1.0, spread=0.2):
        T[name] = (mean + spread * rng.standard_normal(n)).astype(np.float32)
    D = cfg["width"]
    T["embed"] = rng.standard_normal((cfg["vocab"], D)).astype(np.float32)
    bg = (cfg.get("embedding") or {}).get("bigram")
    if bg:
        T["bigram"] = rng.standard_normal((bg["buckets"] + 1, D)).astype(np.float32)
    for i, l in enumerate(cfg["layers"]):
        p, m = f"l{i}.", l["mixer"]
        x = p + "mix."
        vec(p + "norm1", D)
        mat(x + "dq", m["q_rank"], D)
        vec(x + "dq.norm", m["q_rank"])
        mat(x + "uq", m["heads"] * (m["dim"] + m["rot_dim"]), m["q_rank"], gain)
        if "kv_from" not in m:
            mat(x + "dkv", m["kv_rank"] + m["rot_dim"], D)
            vec(x + "dkv.norm", m["kv_rank"])
        mat(x + "uk", m["heads"] * m["dim"], m["kv_rank"], gain)
        mat(x + "uv", m["heads"] * m["vdim"], m["kv_rank"])
        vec(x + "sink", m["heads"], 0.5, 1.5)
        mat(x + "g", m["heads"], D)
        mat(x + "o", D, m["heads"] * m["vdim"])
        if l["mlp"]:
            mat(p + "mlp.gate", l["mlp"]["ff"], D)
            mat(p + "mlp.up", l["mlp"]["ff"], D)
            mat(p + "mlp.down", D, l["mlp"]["ff"])
    vec("final.norm", D)
    mat("head", cfg["vocab"], D)
    return T


def write_folder(path, cfg, tensors):
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    ld.write_safetensors(os.path.join(path, "model.safetensors"), tensors)
    return str(path)


# root mean square over the vocabulary (mean taken off), over the spread of the logits
LIMIT = {"float32": 2e-5, "bfloat16": 0.03}


def logits_error(got, want):
    d = np.asarray(got, dtype=np.float64) - want
    d -= d.mean(axis=-1, keepdims=True)
    return np.sqrt((d * d).mean(axis=-1)) / np.std(want)


def assert_logits(got, want, dtype, what="", factor=1.0):
    e = logits_error(got, want)
    assert np.isfinite(e).all() and e.max() <= factor * LIMIT[dtype], (what, dtype, int(e.argmax()), float(e.max()))


# ---- kernels one by one: structs of the C header, packed tiles --------------------------------------------------------------
def c_struct(name):
    """The ctypes form of a struct in include/m40llm.h."""
    import ctypes as C
    import re
    text = re.sub(r"/\*.*?\*/", "", open(m40.HEADER).read(), flags=re.S)
    body = re.search(r"typedef struct %s \{(.*?)\} %s;" % (name, name), text, flags=re.S).group(1)
    fields = []
    for decl in body.split(";"):
        decl = decl.strip()
        if not decl:
            continue
        ty, names = re.match(r"(?:const\s+)?(\w+)\s*(.*)", decl, flags=re.S).groups()
        for n in names.split(","):
            base = {"uint32_t": C.c_uint32, "uint64_t": C.c_uint64, "float": C.c_float}
            fields.append((n.strip(" *\n"), C.c_void_p if "*" in n else base[ty]))
    return type(name, (C.Structure,), {"_fields_": fields})


def up32(n):
    return (n + 31) // 32 * 32


def as_act(a, dtype):
    """Bits of activations: bf16 (rounded) or f32."""
    return ld.f32_to_bf16(a) if dtype == "bfloat16" else np.ascontiguousarray(a, dtype=np.float32)


def from_act(a, dtype):
    return ld.bf16_to_f32(a) if dtype == "bfloat16" else a


def pack_tiles(a):
    """[N][K] (any dtype) -> 16 x 32 tiles in operand order, zero past the matrix."""
    n, k = a.shape
    N, K = (n + 15) // 16 * 16, up32(k)
    full = np.zeros((N, K), dtype=a.dtype)
    full[:n, :k] = a
    return np.ascontiguousarray(full.reshape(N // 16, 16, K // 32, 4, 8).transpose(0, 2, 3, 1, 4)).reshape(-1)


def unpack_tiles(flat, n, ld_cols):
    N = (n + 15) // 16 * 16
    return flat[:N * ld_cols].reshape(N // 16, ld_cols // 32, 4, 16, 8).transpose(0, 3, 1, 2, 4).reshape(N, ld_cols)[:n]


def close_to(got, want, dtype, scale=None, factor=1.0):
    scale = (np.abs(want).max() or 1.0) if scale is None else scale
    err = np.abs(np.asarray(got, dtype=np.float64) - want).max() / scale
    assert err <= factor * {"float32": 3e-6, "bfloat16": 6e-3}[dtype], float(err)
