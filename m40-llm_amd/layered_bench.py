"""Prefill and decode throughput of layered decoders with random weights beside the framework's closest other model of the same width,
depth and vocabulary.  `bench.py --design NAME` prints what measure() returns: the Pimosun design beside the dense decoder, the Gulidra
design beside Pimosun, whose feed-forward is as wide as the experts a token takes together, the Natatar design beside Gulidra with the same
experts in every layer, the Fomunex design beside Gulidra (dense and routed feed-forwards in turn on both sides) and Natatar.

A case is one shape on one kind of step: a prompt of n tokens run in one step (host clock around the blocking call, the last
token's logits included), or `batch` sequences of `context` tokens that decode greedily from a replayed graph (timed between
full synchronisations).  Cache contents do not change how long a step takes, so contexts are assumed, not computed."""
from __future__ import annotations

import importlib
import time

import numpy as np

pkg = importlib.import_module(__package__)
syn = importlib.import_module(__package__ + ".synthetic")
layered = importlib.import_module(__package__ + ".layered")

BESIDE = dict(pimosun="Pimosun beside the dense decoder", gulidra="Gulidra beside Pimosun", natatar="Natatar beside Gulidra", fomunex="Fomunex beside Gulidra and Natatar")
SHAPES = {
    # name: layered decoder, and the dense decoder's heads at the same width
    "2k": dict(width=2048, heads=16, dim=128, rot_dim=64, vdim=128, kv_rank=512, q_rank=768, ff=5632, vocab=32000, layers=8, kv_heads=2),
    "4k": dict(width=4096, heads=32, dim=128, rot_dim=64, vdim=128, kv_rank=512, q_rank=1536, ff=11008, vocab=32000, layers=4, kv_heads=8),
}
PREFILL = (512, 4096)
DECODE = ((1, 1024), (8, 4096), (32, 4096))


def pimosun_config(s: dict) -> dict:
    rot = dict(base=10000.0, dims=s["rot_dim"], scaling=dict(factor=8.0, original=4096, fast=32.0, slow=1.0))
    mixer = dict(heads=s["heads"], dim=s["dim"], rot_dim=s["rot_dim"], vdim=s["vdim"], kv_rank=s["kv_rank"], q_rank=s["q_rank"],
                 scale=float((s["dim"] + s["rot_dim"]) ** -0.5), rot=rot)
    half = s["layers"] // 2
    layers = [dict(type="latent_attention", mixer=dict(mixer, **({"kv_from": half - 1} if i >= half else {})), mlp=dict(kind="dense", ff=s["ff"]))
              for i in range(s["layers"])]
    return dict(architecture="Pimosun", vocab=s["vocab"], width=s["width"], norm=dict(eps=1e-5),
                embedding=dict(bigram=dict(buckets=20011, mul_prev=31, mul_cur=7)), layers=layers)


# Gulidra at Pimosun's sizes: half of the layers routed, one in four a lightning layer, the second half of the attention layers reading the first
# half's keys; a token's experts together are as wide as the dense feed-forward
GULIDRA = {
    "2k": dict(kv_heads=4, dim=64, conv=4, experts=32, identity=2, top=4, expert_ff=1408, light=(16, 128, 128)),
    "4k": dict(kv_heads=8, dim=64, conv=4, experts=32, identity=2, top=4, expert_ff=2752, light=(32, 128, 128)),
}


def gulidra_config(name: str, routed=False) -> dict:
    """routed: experts in every layer, none of them the identity."""
    s, g = SHAPES[name], GULIDRA[name]
    mixer = dict(heads=s["heads"], kv_heads=g["kv_heads"], dim=g["dim"], vdim=s["vdim"], conv=g["conv"], diff=0.3, scale=float(g["dim"] ** -0.5))
    heads, dim, vdim = g["light"]
    light = dict(heads=heads, dim=dim, vdim=vdim, decay=[float(1 - 2.0 ** -(2 + 8 * i / heads)) for i in range(heads)])
    moe = dict(kind="moe", expert=dict(ff=g["expert_ff"]), router=dict(experts=g["experts"], identity=g["identity"], top=g["top"]))
    if routed:
        moe["router"]["identity"] = 0
    dense = moe if routed else dict(kind="dense", ff=s["ff"])
    layers = []
    for i in range(s["layers"]):
        mlp = moe if i % 2 else dense
        if i % 4 == 3:
            layers.append(dict(type="lightning", mixer=light, mlp=mlp))
        else:
            layers.append(dict(type="attention", mixer=dict(mixer, **({"kv_from": i - 2} if i % 4 == 2 else {})), mlp=mlp))
    return dict(architecture="Gulidra", vocab=s["vocab"], width=s["width"], norm=dict(eps=1e-5), embedding=dict(scale=1.0), residual_mult=0.7,
                max_positions=8192, layers=layers)


# Natatar at the same sizes: of four layers one with attention beside a matrix memory, two of attention, one of the delta rule; four streams
NATATAR = {
    "2k": dict(streams=4, kv_heads=4, dim=128, conv=4, experts=32, top=4, expert_ff=1408, groups=(8, 4), memory=(16, 128, 128), delta=(16, 16, 128, 128)),
    "4k": dict(streams=4, kv_heads=8, dim=128, conv=4, experts=32, top=4, expert_ff=2752, groups=(8, 4), memory=(32, 128, 128), delta=(32, 32, 128, 128)),
}


def natatar_config(name: str) -> dict:
    s, g = SHAPES[name], NATATAR[name]
    mixer = dict(heads=s["heads"], kv_heads=g["kv_heads"], dim=g["dim"], vdim=s["vdim"], scale=float(g["dim"] ** -0.5))
    rot = dict(base=500000.0, dims=g["dim"], scaling=dict(factor=8.0, original=4096, fast=32.0, slow=1.0))
    h, d, v = g["memory"]
    parallel = dict(left=dict(mixer, rot=rot), left_scale=0.7, right=dict(heads=h, dim=d, vdim=v, gate_cap=12.0), right_scale=1.1)
    h, k, d, v = g["delta"]
    delta = dict(heads=h, kv_heads=k, dim=d, vdim=v, conv=g["conv"])
    kinds = [dict(type="parallel", mixer=parallel), dict(type="attention", mixer=dict(mixer, v_mix=True)), dict(type="channel_delta", mixer=delta),
             dict(type="attention", mixer=dict(mixer, v_mix=True))]
    moe = dict(kind="moe", expert=dict(ff=g["expert_ff"]), router=dict(experts=g["experts"], top=g["top"], scale=2.0, groups=dict(count=g["groups"][0], keep=g["groups"][1])))
    return dict(architecture="Natatar", vocab=s["vocab"], width=s["width"], streams=g["streams"], norm=dict(eps=1e-5), embedding=dict(scale=1.0), residual_mult=0.3,
                layers=[dict(kinds[i % 4], mlp=moe) for i in range(s["layers"])])


# Fomunex at the same sizes: of four layers two of attention (a window of 1024 tokens, one of all positions), one of time mixing, one state space layer;
# dense and routed feed-forwards in turn, the dense one without a gate, so wider by half for the same weights
FOMUNEX = {
    "2k": dict(kv_heads=4, dim=128, windows=(1024, 8192), mixing=(32, 64), space=(64, 8, 128, 64, 4, 8), ff=8448, experts=32, top=4, expert_ff=1408),
    "4k": dict(kv_heads=8, dim=128, windows=(1024, 8192), mixing=(64, 64), space=(128, 8, 128, 64, 4, 8), ff=16512, experts=32, top=4, expert_ff=2752),
}


def fomunex_config(name: str) -> dict:
    s, g = SHAPES[name], FOMUNEX[name]
    attention = [dict(type="attention", mixer=dict(heads=s["heads"], kv_heads=g["kv_heads"], dim=g["dim"], vdim=s["vdim"], mask=dict(size=w), softcap=30.0,
                                                   scale=float(g["dim"] ** -0.5))) for w in g["windows"]]
    h, d = g["mixing"]
    mixing = dict(type="wkv", mixer=dict(heads=h, dim=d))
    space = dict(type="mamba2", mixer=dict(zip(("heads", "groups", "state", "vdim", "conv", "norm_groups"), g["space"])))
    moe = dict(kind="moe", expert=dict(ff=g["expert_ff"], limit=7.0), router=dict(experts=g["experts"], top=g["top"]))
    dense = dict(kind="dense", ff=g["ff"])
    kinds = [dict(attention[0], mlp=dense), dict(mixing, mlp=moe), dict(attention[1], mlp=dense), dict(space, mlp=moe)]
    return dict(architecture="Fomunex", vocab=s["vocab"], width=s["width"], norm=dict(eps=1e-5), max_positions=8192, logit_scale=0.5, logit_softcap=30.0,
                layers=[kinds[i % 4] for i in range(s["layers"])])


def layer_flops_per_token(s: dict, own: bool) -> float:
    """Matrix-product flops of one layer and token outside attention's own products (keys and values from the latent included)."""
    w, h = s["width"], s["heads"]
    n = w * (s["q_rank"] + h) + s["q_rank"] * h * (s["dim"] + s["rot_dim"]) + h * (s["dim"] + s["vdim"]) * s["kv_rank"] + h * s["vdim"] * w + 3 * w * s["ff"]
    return 2.0 * (n + (w * (s["kv_rank"] + s["rot_dim"]) if own else 0))


def layered_cases(ctx, s, prefill=PREFILL, decode=DECODE, reps=3, steps=32, warmup=4, cfg=None):
    out = {}
    cfg = cfg or pimosun_config(s)
    rng = np.random.default_rng(0)
    slots = max([b for b, _ in decode] + [1])
    tokens = max([b * (c + steps + warmup + 64) for b, c in decode] + [n + 64 for n in prefill])
    m = layered.LayeredModel.random(ctx, cfg, seed=1, std=0.02, max_tokens=tokens, max_sequences=slots, max_rows=max(list(prefill) + [64]))
    m.set_tie_guard(-1.0)
    for n in prefill:
        prompt = rng.integers(0, s["vocab"], size=n).astype(np.uint32)
        best = None
        for r in range(reps + 1):
            t0 = time.perf_counter()
            m.step([(0, prompt, [n - 1])])
            ms = (time.perf_counter() - t0) * 1e3
            m.release(0)
            if r and (best is None or ms < best):
                best = ms
        out[f"prefill {n}"] = dict(ms=best, tok_s=n / (best * 1e-3))
    for b, c in decode:
        for i in range(b):
            m.assume_length(i, c)
        first = rng.integers(0, s["vocab"], size=b)
        _, ms = m.decode_batch_timed(np.arange(b), np.full(b, c), first, warmup, steps)
        for i in range(b):
            m.release(i)
        out[f"decode {b} x {c}"] = dict(ms=ms / steps, tok_s=b * steps / (ms * 1e-3))
    m.close()
    return out


def dense_cases(ctx, s, prefill=PREFILL, decode=DECODE, reps=3, steps=32, warmup=4):
    out = {}
    cfg = dict(syn.TINYLLAMA_1B, n_layers=s["layers"], d_model=s["width"], q_heads=s["heads"], kv_heads=s["kv_heads"],
               head_dim=s["width"] // s["heads"], ffn=s["ff"], vocab=s["vocab"])
    W = syn.make_weights(cfg, seed=0, unique_layers=1, tie_embeddings=True)
    rng = np.random.default_rng(0)
    slots = max([b for b, _ in decode] + [1])
    length = max([c + steps + warmup + 8 for _, c in decode] + [n + 8 for n in prefill])
    dm = syn.DeviceModel(ctx, cfg, W, max_seq_len=length, max_sequences=slots)
    dm.set_mode(2)
    dm.H.m40host_model_set_tie_guard(dm.h, -1.0)
    for n in prefill:
        prompt = rng.integers(0, s["vocab"], size=n).tolist()
        best = None
        for r in range(reps + 1):
            t0 = time.perf_counter()
            dm.forward_prefill([0], [prompt])
            ms = (time.perf_counter() - t0) * 1e3
            if r and (best is None or ms < best):
                best = ms
        out[f"prefill {n}"] = dict(ms=best, tok_s=n / (best * 1e-3))
    for b, c in decode:
        k = rng.standard_normal((c, cfg["kv_heads"], cfg["head_dim"]), dtype=np.float32).astype(np.float16).view(np.uint16)
        dk = ctx.to_device(k)
        for i in range(b):
            for l in range(cfg["n_layers"]):
                pkg.check(ctx.lib.m40llm_ext_kvcache_bulk_fill_f16(ctx.h, dm.kv_handle(), dm.H.m40host_model_kv_slot(dm.h, i, l), dk.ptr, dk.ptr, c),
                          "m40llm_ext_kvcache_bulk_fill_f16")
        try:
            _, ms = dm.decode_batch_timed(np.arange(b), np.full(b, c), rng.integers(0, s["vocab"], size=b), warmup, steps)
            out[f"decode {b} x {c}"] = dict(ms=ms / steps, tok_s=b * steps / (ms * 1e-3))
        except RuntimeError as e:
            out[f"decode {b} x {c}"] = dict(error=str(e))
        dk.free()
    dm.close()
    return out


def measure(ctx, shapes=None, steps=32, warmup=4, dense=True, design="pimosun") -> dict:
    out = {}
    if design == "fomunex":
        for name in shapes or SHAPES:
            s = SHAPES[name]
            out[name] = {"shape": dict(s, **FOMUNEX[name]), "fomunex": layered_cases(ctx, s, steps=steps, warmup=warmup, cfg=fomunex_config(name)),
                         "gulidra": layered_cases(ctx, s, steps=steps, warmup=warmup, cfg=gulidra_config(name)),
                         "natatar": layered_cases(ctx, s, steps=steps, warmup=warmup, cfg=natatar_config(name))}
        return out
    if design == "natatar":
        for name in shapes or SHAPES:
            s = SHAPES[name]
            out[name] = {"shape": dict(s, **NATATAR[name]), "natatar": layered_cases(ctx, s, steps=steps, warmup=warmup, cfg=natatar_config(name)),
                         "gulidra": layered_cases(ctx, s, steps=steps, warmup=warmup, cfg=gulidra_config(name, routed=True))}
        return out
    if design == "gulidra":
        for name in shapes or SHAPES:
            s = SHAPES[name]
            out[name] = {"shape": dict(s, **GULIDRA[name]), "gulidra": layered_cases(ctx, s, steps=steps, warmup=warmup, cfg=gulidra_config(name)),
                         "pimosun": layered_cases(ctx, s, steps=steps, warmup=warmup)}
        return out
    for name in shapes or SHAPES:
        s = SHAPES[name]
        out[name] = {"shape": {k: v for k, v in s.items() if k != "kv_heads"}, "pimosun": layered_cases(ctx, s, steps=steps, warmup=warmup)}
        if dense:
            out[name]["dense_kv_heads"] = s["kv_heads"]
            out[name]["dense"] = dense_cases(ctx, s, steps=steps, warmup=warmup)
    return out
