"""The Gulidra design without a device: its reader (through tests/layered_host_check.cpp) and the plain restatement against itself."""
import copy

import numpy as np
import pytest

from gulidra_common import CONFIGS, od, random_tensors, write_folder
from test_layered_host import check, written  # noqa: F401  (check is a fixture)


@pytest.mark.parametrize("name", list(CONFIGS))
def test_the_design_is_read_from_its_configuration(check, tmp_path, name):  # noqa: F811
    cfg = CONFIGS[name]()
    got = check("spec", written(tmp_path, cfg))
    assert (got["architecture"], got["vocab"], got["width"], got["positions"]) == ("Gulidra", cfg["vocab"], cfg["width"], cfg["max_positions"])
    for key, want in (("eps", cfg["norm"]["eps"]), ("embedding_scale", cfg["embedding"]["scale"]), ("residual_mult", cfg["residual_mult"])):
        assert abs(got[key] - want) < 1e-6 * want
    assert len(got["layers"]) == len(cfg["layers"])
    for g, l in zip(got["layers"], cfg["layers"]):
        m = l["mixer"]
        if l["type"] == "attention":
            assert g["sizes"] == [m["heads"], m["kv_heads"], m["dim"], m["vdim"], m.get("conv", 0)]
            assert g["kv_from"] == m.get("kv_from", -1) and g["diff"] == m["diff"] and abs(g["scale"] - m["scale"]) < 1e-6 * m["scale"]
        else:
            assert g["sizes"] == [m["heads"], m["dim"], m["vdim"]] and g["decay"] == m["decay"]
        f = l["mlp"]
        assert g["ff"] == (f["ff"] if f and f["kind"] == "dense" else 0) and g["silu"] == (g["ff"] > 0)
        if f and f["kind"] == "moe":
            r = f["router"]
            assert g["experts"] == [r["experts"], r["identity"], r["top"], f["expert"]["ff"]]
        else:
            assert "experts" not in g


def test_bad_configurations_are_refused(check, tmp_path):  # noqa: F811
    def error(change):
        cfg = copy.deepcopy(CONFIGS["odd"]())
        change(cfg["layers"], cfg)
        return check("spec", written(tmp_path, cfg)).get("error", "")
    assert "unknown mixer" in error(lambda L, c: L[0].update(type="latent_attention"))
    assert "unknown feed-forward" in error(lambda L, c: L[0]["mlp"].update(kind="sparse"))
    assert "size is zero" in error(lambda L, c: L[0]["mixer"].update(vdim=0))
    assert "size is zero" in error(lambda L, c: L[1]["mixer"].update(dim=0))
    assert "size is zero" in error(lambda L, c: L[0]["mlp"]["expert"].update(ff=0))
    assert "multiple of kv_heads" in error(lambda L, c: L[0]["mixer"].update(heads=5))
    assert "one number a head" in error(lambda L, c: L[1]["mixer"]["decay"].pop())
    assert "positive" in error(lambda L, c: L[1]["mixer"].update(decay=[0.5, 0.0, 0.9]))
    assert "earlier layer" in error(lambda L, c: L[0]["mixer"].update(kv_from=0))
    for change in (lambda L, c: L[3]["mixer"].update(kv_from=1),               # not an attention layer
                   lambda L, c: L[5]["mixer"].update(kv_from=3),               # reads another layer's itself
                   lambda L, c: L[3]["mixer"].update(dim=24), lambda L, c: L[3]["mixer"].update(vdim=36), lambda L, c: L[3]["mixer"].update(kv_heads=4)):
        assert "keys of its own and the same" in error(change)
    assert "router.top" in error(lambda L, c: L[0]["mlp"]["router"].update(top=11))
    assert "missing key 'diff'" in error(lambda L, c: L[0]["mixer"].pop("diff"))
    assert "missing key 'max_positions'" in error(lambda L, c: c.pop("max_positions"))
    # what may be left out
    cfg = copy.deepcopy(CONFIGS["odd"]())
    for k in ("embedding", "residual_mult"):
        cfg.pop(k)
    cfg["layers"][0]["mlp"]["router"].pop("identity")
    got = check("spec", written(tmp_path, cfg))
    assert (got["embedding_scale"], got["residual_mult"], got["layers"][0]["experts"][1]) == (1, 1, 0)


def test_restatement_portions_equal_whole(tmp_path):
    for name in CONFIGS:
        cfg = CONFIGS[name]()
        m = od.Model.load(write_folder(tmp_path / name, cfg, random_tensors(cfg, 5)))
        t = np.random.default_rng(2).integers(0, cfg["vocab"], size=23).tolist()
        s = m.sequence()
        whole = s.feed(t)
        u = m.sequence()
        parts = np.concatenate([u.feed(t[a:b]) for a, b in ((0, 1), (1, 3), (3, 20), (20, 23))])
        assert np.abs(whole - parts).max() < 1e-9 * np.abs(whole).max()
        assert np.allclose(s.margins, u.margins)


def test_choice_margin():
    z = np.array([[2.0, 1.0, 0.0], [0.0, 1.0, 2.0]])
    w = np.eye(3)
    m = od.choice_margin(z, w, np.zeros(3), 1)
    assert np.allclose(m, 1 - np.exp(-1.0))
    s = np.exp(z) / np.exp(z).sum(axis=1, keepdims=True)
    c = np.array([0.0, s[0, 0] - s[0, 1] + 1e-9, 0.0])
    assert od.choice_margin(z, w, c, 1)[0] < 1e-8 and np.isinf(od.choice_margin(z, w, c, 3)).all()


def test_restatement_notices_planted_mistakes():
    """Each mistake, planted in the restatement, moves its logits far beyond what the device comparisons allow."""
    cfg = CONFIGS["odd"]()
    T = random_tensors(cfg, 3)
    t = np.random.default_rng(2).integers(0, cfg["vocab"], size=90).tolist()
    base = od.Model(cfg, T).sequence().feed(t)

    def moved(change=lambda c, U: None, feed=None, **planted):
        c, U = copy.deepcopy(cfg), {k: v.copy() for k, v in T.items()}
        change(c, U)
        kept = {k: getattr(od, k) for k in planted}
        try:
            for k, f in planted.items():
                setattr(od, k, f)
            s = od.Model(c, U).sequence()
            d = (feed(s) if feed else s.feed(t)) - base
        finally:
            for k, f in kept.items():
                setattr(od, k, f)
        d -= d.mean(axis=1, keepdims=True)
        return np.sqrt((d * d).mean(axis=1)).max() / np.std(base)

    def lose(key):
        def feed(s):
            a = s.feed(t[:40])
            for st in s.state:
                for k in list(st):
                    if k.endswith(key):
                        st[k] = np.zeros_like(st[k])
            return np.concatenate([a, s.feed(t[40:])])
        return feed

    def mixers(**kw):
        return lambda c, U: [l["mixer"].update({k: f(l["mixer"][k]) for k, f in kw.items() if k in l["mixer"]}) for l in c["layers"]]
    def own_keys(c, U):                 # layer 0's projections, but of layer 3's input
        c["layers"][3]["mixer"].pop("kv_from")
        for k in ("k", "v", "k.conv", "v.conv", "k.norm"):
            U["l3.mix." + k] = T["l0.mix." + k]

    def shifted(h, w, c, top):
        chosen, weight = route(h, w, c, top)
        return chosen, weight + c[chosen]
    route, join, conv, attend = od.route, od.join_maps, od.short_convolution, od.softmax_attend
    mistakes = dict(
        state=dict(feed=lose("S")), convolution_state=dict(feed=lose(".v")), query_convolution_state=dict(feed=lose(".q")),
        scale=dict(change=mixers(scale=lambda v: v * 1.1)), diff=dict(change=mixers(diff=lambda v: v + 0.02)),
        decay=dict(change=mixers(decay=lambda v: [d * 0.99 for d in v])),
        own_keys=dict(change=own_keys),
        positions=dict(change=lambda c, U: U.update(pos=np.roll(U["pos"], 1, axis=0))), embedding=dict(change=lambda c, U: c["embedding"].update(scale=1.0)),
        eps=dict(change=lambda c, U: c["norm"].update(eps=0.0)), residual=dict(change=lambda c, U: c.update(residual_mult=1.0)),
        correction=dict(change=lambda c, U: [U.update({k: v * 0}) for k, v in T.items() if k.endswith("correction")]),
        gate=dict(change=lambda c, U: [U.update({k: v * 0}) for k, v in T.items() if k.endswith("mix.g")]),
        no_norm_of_the_difference=dict(join_maps=lambda a1, a2, lam, diff, eps: (a1 - lam * a2) * (1 - diff)),
        second_map_added=dict(join_maps=lambda a1, a2, lam, diff, eps: join(a1, -a2, lam, diff, eps)),
        one_key_late=dict(softmax_attend=lambda q, k, v, s, p: attend(q, k, v, s, np.maximum(np.asarray(p) - 1, 0))),
        taps_reversed=dict(short_convolution=lambda u, b, w: conv(u, b, w[:, ::-1])),
        weights_with_the_correction=dict(route=shifted))
    for name, m in mistakes.items():
        assert moved(**m) > 2e-3, name           # a hundred times the 32-bit limit
    assert moved() == 0
