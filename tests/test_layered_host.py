"""Host side of layered decoders without a device: reading a design from config.json, rotation constants, safetensors, the page pool
and the scheduler's mixed steps (through tests/layered_host_check.cpp), and the plain restatement against itself."""
import copy
import json
import os
import subprocess

import numpy as np
import pytest

from pimosun_common import CONFIGS, ld, mixer, random_tensors, write_folder

HERE = os.path.dirname(os.path.abspath(__file__))


@pytest.fixture(scope="module")
def check(tmp_path_factory):
    exe = str(tmp_path_factory.mktemp("host") / "check")
    subprocess.run(["g++", "-O1", "-std=c++17", "-Wall", "-I", os.path.join(HERE, "..", "include"), os.path.join(HERE, "layered_host_check.cpp"), "-o", exe,
                    "-lpthread"], check=True)

    def run(*words):
        out = subprocess.run([exe], input=" ".join(str(w) for w in words) + "\n", capture_output=True, text=True, check=True).stdout
        return json.loads(out)
    return run


def written(tmp_path, cfg, name="config.json"):
    p = tmp_path / name
    p.write_text(cfg if isinstance(cfg, str) else json.dumps(cfg))
    return str(p)


@pytest.mark.parametrize("name", list(CONFIGS))
def test_a_design_is_read_from_its_configuration(check, tmp_path, name):
    cfg = CONFIGS[name]()
    got = check("spec", written(tmp_path, cfg))
    assert (got["architecture"], got["vocab"], got["width"]) == ("Pimosun", cfg["vocab"], cfg["width"])
    assert abs(got["eps"] - cfg["norm"]["eps"]) < 1e-6 * cfg["norm"]["eps"]
    assert got["bigram"] == cfg["embedding"].get("bigram", {}).get("buckets", -1)
    for g, l in zip(got["layers"], cfg["layers"]):
        m = l["mixer"]
        assert g["sizes"] == [m[k] for k in ("heads", "dim", "rot_dim", "vdim", "kv_rank", "q_rank")]
        assert g["kv_from"] == m.get("kv_from", -1) and g["ff"] == (l["mlp"]["ff"] if l["mlp"] else 0)
        assert abs(g["scale"] - m["scale"]) < 1e-6 * m["scale"]
        f, mag = ld.rotation(m["rot"])
        assert np.allclose(g["freq"], f, rtol=1e-14) and abs(g["magnitude"] - mag) < 1e-14
    assert len(got["layers"]) == len(cfg["layers"])


@pytest.mark.parametrize("scaling", [None, dict(factor=40.0, original=4096, fast=32, slow=1), dict(factor=4.0, original=16, fast=64.0, slow=0.01),
                                     dict(factor=2.5, original=1000, fast=3.0, slow=3.0), dict(factor=1.0, original=512, fast=8.0, slow=2.0)])
@pytest.mark.parametrize("dims,base", [(2, 10.0), (16, 1e4), (64, 5e6)])
def test_rotation_frequencies(check, tmp_path, scaling, dims, base):
    cfg = CONFIGS["one"]()
    cfg["layers"][0]["mixer"] = mixer(1, 4, dims, 4, 4, 4, base, scaling)
    got = check("spec", written(tmp_path, cfg))["layers"][0]
    f, mag = ld.rotation(cfg["layers"][0]["mixer"]["rot"])
    assert np.allclose(got["freq"], f, rtol=1e-13) and abs(got["magnitude"] - mag) < 1e-13


def test_bad_configurations_are_refused(check, tmp_path):
    def error(change):
        cfg = copy.deepcopy(CONFIGS["odd"]())
        change(cfg)
        return check("spec", written(tmp_path, cfg)).get("error", "")
    L = lambda cfg, i: cfg["layers"][i]
    assert "unknown architecture" in error(lambda c: c.update(architecture="Nothing"))
    assert "unknown mixer" in error(lambda c: L(c, 0).update(type="other"))
    assert "unknown feed-forward" in error(lambda c: L(c, 0)["mlp"].update(kind="sparse"))
    assert "size is zero" in error(lambda c: L(c, 0)["mixer"].update(heads=0))
    assert "earlier layer" in error(lambda c: L(c, 0)["mixer"].update(kv_from=0))
    assert "kv_from" in error(lambda c: L(c, 3)["mixer"].update(kv_from=2))          # a layer that reads another's entries itself
    assert "kv_from" in error(lambda c: L(c, 2)["mixer"].update(kv_rank=41))
    assert "kv_from" in error(lambda c: L(c, 2)["mixer"]["rot"].update(base=3.0))
    assert "rot.dims" in error(lambda c: L(c, 1)["mixer"]["rot"].update(dims=7))
    assert "missing key 'vocab'" in error(lambda c: c.pop("vocab"))
    assert "not a 32-bit count" in error(lambda c: c.update(width=2.5))
    for text in ("", "{", '{"a": 1,}', "[1, 2", '{"a" 1}', "nul", '{"a": 1} x'):
        assert check("spec", written(tmp_path, text)).get("error")


def test_safetensors_reader(check, tmp_path):
    p = str(tmp_path / "t.safetensors")
    v = np.arange(-6, 6, dtype=np.float32).reshape(3, 4)
    ld.write_safetensors(p, {"a.b": v, "c": v[0] * 0.5})
    assert check("tensors", p, "a.b", 3, 4) == v.reshape(-1).tolist()
    assert check("tensors", p, "c", 4) == (v[0] * 0.5).tolist()
    assert "another shape" in check("tensors", p, "a.b", 4, 3)["error"]
    assert "no tensor" in check("tensors", p, "d", 4)["error"]
    raw = open(p, "rb").read()
    for bad in (raw[:4], raw[:20], raw[:-3], b"\xff" * 8 + raw[8:]):
        q = str(tmp_path / "bad.safetensors")
        open(q, "wb").write(bad)
        assert check("tensors", q, "a.b", 3, 4)["error"]


def test_page_pool_gives_back_and_keeps_promises(check):
    r = check("pages", 6, 64, 3, "g 0 1 g 0 64 g 0 65 a 0 65 7 g 1 256 g 1 257 f 0 g 1 257 a 1 200 9 f 1 f 1 g 5 1")
    assert [x["free"] for x in r] == [5, 5, 4, 4, 0, 0, 2, 1, 1, 6, 6, 6]
    assert r[5]["result"] == "the cache pool has no page left" and len(r[5]["pages"]) == 4
    assert (r[3]["length"], r[3]["prev"]) == (65, 7) and (r[6]["length"], r[6]["prev"], r[6]["pages"]) == (0, 0xffffffff, [])
    assert set(r[4]["pages"]) | set(r[2]["pages"]) == set(range(6))
    assert "out of range" in r[11]["result"]
    # pages promised to one sequence are not given to another, and come back with it
    r = check("pages", 4, 64, 2, "r 0 192 g 1 64 g 1 65 r 1 128 g 0 100 g 0 192 f 0 g 1 256")
    assert [x["result"] for x in r] == [True, True, "the cache pool has no page left", False, True, True, True, True]
    assert [x["free"] for x in r] == [4, 3, 3, 3, 1, 0, 3, 0]


def test_scheduler_steps_mix_portions_and_tokens(check):
    r = check("scheduler", 6, 64, 3, "p 4 3 p 13 2 p 1 4 p 9 1")
    for i, (n, m) in enumerate(((4, 3), (13, 2), (1, 4), (9, 1))):
        q = r["requests"][i]
        assert q["state"] == 3 and q["ids"] == [(10 * i + n + k) % 50 for k in range(m)], q
    assert r["free"] == 16
    assert r["ticks"][0] == [[0, 0, 4, 1], [1, 0, 2, 0]]               # as much of the second prompt as the tick still takes
    assert r["ticks"][1] == [[0, 4, 1, 1], [1, 2, 5, 0]]               # a decoded token beside its next portion
    assert all(sum(x[2] for x in t) <= 6 for t in r["ticks"])
    # every portion of a prompt continues where the one before ended
    at = {}
    for t in r["ticks"]:
        for slot, start, n, _ in t:
            assert start in (0, at.get(slot, 0))
            at[slot] = start + n


def test_scheduler_waits_for_pages_and_refuses_nothing_that_fits(check):
    # 16 pages of 4 tokens; each request may grow to 32 tokens: two fit at a time, in order of arrival
    r = check("scheduler", 100, 64, 4, "p 20 12 p 20 12 p 20 12 p 2 2")
    assert [q["state"] for q in r["requests"]] == [3, 3, 3, 3] and r["free"] == 16
    assert [x[0] for x in r["ticks"][0]] == [0, 1]
    r = check("scheduler", 100, 64, 1, "p 60 9")
    assert r["requests"][0]["state"] == 5 and "context window" in r["requests"][0]["error"] and len(r["requests"][0]["ids"]) == 5


# ---- the restatement itself -----------------------------------------------------------------------------------------------
def test_restatement_portions_equal_whole(tmp_path):
    for name in CONFIGS:
        cfg = CONFIGS[name]()
        folder = write_folder(tmp_path / name, cfg, random_tensors(cfg, 5))
        m = ld.Model.load(folder)
        t = np.random.default_rng(2).integers(0, cfg["vocab"], size=23).tolist()
        whole = m.sequence().feed(t)
        s = m.sequence()
        parts = np.concatenate([s.feed(t[a:b]) for a, b in ((0, 1), (1, 3), (3, 20), (20, 23))])
        assert np.abs(whole - parts).max() < 1e-9 * np.abs(whole).max()


def test_restatement_notices_planted_mistakes(tmp_path):
    """Each mistake, planted in the restatement, moves its logits far beyond what the device comparisons allow."""
    cfg = CONFIGS["odd"]()
    T = random_tensors(cfg, 3)
    t = np.random.default_rng(2).integers(0, cfg["vocab"], size=90).tolist()
    base = ld.Model(cfg, T).sequence().feed(t)

    def moved(change):
        c, U = copy.deepcopy(cfg), {k: v.copy() for k, v in T.items()}
        change(c, U)
        d = ld.Model(c, U).sequence().feed(t) - base
        d -= d.mean(axis=1, keepdims=True)
        return np.sqrt((d * d).mean(axis=1)).max() / np.std(base)

    def no_sink(c, U):
        for k in U:
            if k.endswith(".sink"):
                U[k][:] = -1e4

    def rot(key, value):
        def f(c, U):
            for l in c["layers"]:
                l["mixer"]["rot"].get("scaling", {}).update({key: value}) if key in ("factor", "original", "fast") else l["mixer"]["rot"].update({key: value})
        return f

    def own_entries(c, U):
        c["layers"][2]["mixer"].pop("kv_from")
        U["l2.mix.dkv"], U["l2.mix.dkv.norm"] = U["l0.mix.dkv"], U["l0.mix.dkv.norm"]
    for change in (no_sink, rot("base", 501.0), rot("factor", 5.0), rot("original", 80), own_entries,
                   lambda c, U: c["norm"].update(eps=0.0), lambda c, U: c["embedding"]["bigram"].update(mul_prev=12),
                   lambda c, U: [l["mixer"].update(scale=l["mixer"]["scale"] * 1.1) for l in c["layers"]],
                   lambda c, U: [U.update({k: v * 0.0}) for k, v in U.items() if k.endswith("mix.g")]):
        assert moved(change) > 2e-3, change          # a hundred times the 32-bit limit
