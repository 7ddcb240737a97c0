"""The Fomunex design without a device: its reader (through tests/layered_host_check.cpp) and the plain restatement against itself."""
import copy

import numpy as np
import pytest

from fomunex_common import CONFIGS, pd, random_config, random_tensors, write_folder
from test_layered_host import check, written  # noqa: F401  (check is a fixture)


def near(a, b):
    return abs(a - b) <= 1e-6 * abs(b)


@pytest.mark.parametrize("name", list(CONFIGS) + [0, 1, 2, 3])
def test_the_design_is_read_from_its_configuration(check, tmp_path, name):  # noqa: F811
    cfg = random_config(name) if isinstance(name, int) else CONFIGS[name]()
    got = check("spec", written(tmp_path, cfg))
    assert (got["architecture"], got["vocab"], got["width"], got["streams"], got["positions"]) == ("Fomunex", cfg["vocab"], cfg["width"], 1, cfg["max_positions"])
    assert got["norm_scalar"] and not got["tied_head"] and not got["around_zero"] and got["bigram"] == -1 and got["embedding_scale"] == 1 and got["residual_mult"] == 1
    assert near(got["eps"], cfg["norm"]["eps"]) and near(got["logits"][0], cfg["logit_scale"]) and near(got["logits"][1], cfg["logit_softcap"])
    assert len(got["layers"]) == len(cfg["layers"])
    for i, (g, l) in enumerate(zip(got["layers"], cfg["layers"])):
        m = l["mixer"]
        assert g["tensors_of"] == (pd.tensors_of(cfg["layers"], i) if "weights_of" in l else -1)
        if l["type"] == "attention":
            assert g["sizes"] == [m[k] for k in ("heads", "kv_heads", "dim", "vdim")] and near(g["scale"], m["scale"]) and g["flags"] == [0, 0, 0, 0]
            assert g["scores"][:3] == [1, 1, 1] and near(g["scores"][3], m["softcap"]) and g["scores"][4] == m["mask"]["size"] and "freq" not in g
        elif l["type"] == "wkv":
            assert g["sizes"] == [m["heads"], m["dim"]]
        else:
            assert g["sizes"] == [m[k] for k in ("heads", "groups", "state", "vdim", "conv", "norm_groups")]
        f = l["mlp"]
        assert g["ff"] == 0 and g.get("poly") == (f["ff"] if f and f["kind"] == "dense" else None) and ("experts" in g) == bool(f and f["kind"] == "moe")
        if f and f["kind"] == "moe":
            assert g["experts"] == [f["router"]["experts"], 0, f["router"]["top"], f["expert"]["ff"]] and not g["correction"] and g["sigmoid"] and g["weight_input"]
            assert near(g["limit"][0], f["expert"]["limit"]) and near(g["limit"][1], 1.702) and g["activation"] == 2 and g["groups"] == [1, 1] and g["router_scale"] == 1


def test_bad_configurations_are_refused(check, tmp_path):  # noqa: F811
    def error(change):
        cfg = copy.deepcopy(CONFIGS["odd"]())
        change(cfg["layers"], cfg)
        return check("spec", written(tmp_path, cfg)).get("error", "")
    assert error(lambda L, c: None) == ""
    assert "unknown mixer" in error(lambda L, c: L[3].update(type="lightning"))
    assert "unknown feed-forward" in error(lambda L, c: L[1]["mlp"].update(kind="sparse"))
    for i, key in ((3, "vdim"), (1, "dim"), (9, "conv"), (9, "state"), (10, "norm_groups"), (10, "groups")):
        assert "size is zero" in error(lambda L, c: L[i]["mixer"].update({key: 0}))
    assert "size is zero" in error(lambda L, c: L[1]["mlp"].update(ff=0))
    assert "multiple of kv_heads" in error(lambda L, c: L[3]["mixer"].update(heads=5))
    assert "multiple of groups" in error(lambda L, c: L[9]["mixer"].update(groups=2))
    assert "norm_groups" in error(lambda L, c: L[10]["mixer"].update(norm_groups=5))
    assert "scale is zero" in error(lambda L, c: L[3]["mixer"].update(scale=0))
    assert "softcap" in error(lambda L, c: L[3]["mixer"].update(softcap=-1))
    assert "mask.size" in error(lambda L, c: L[3]["mixer"]["mask"].update(size=0))
    assert "expert.limit" in error(lambda L, c: [L[i]["mlp"]["expert"].update(limit=-1) for i in (4, 6, 8)])
    assert "router.top" in error(lambda L, c: [L[i]["mlp"]["router"].update(top=6) for i in (4, 6, 8)])
    for change in (lambda L, c: L[5].update(weights_of=5), lambda L, c: L[5].update(weights_of=11), lambda L, c: L[6].update(weights_of=8)):
        assert "tensors of its own" in error(change)
    for change in (lambda L, c: L[5].update(weights_of=9), lambda L, c: L[5].update(mlp=None), lambda L, c: L[7]["mixer"].update(softcap=9.5)):
        assert "same kind and sizes" in error(change)
    assert "missing key 'max_positions'" in error(lambda L, c: c.pop("max_positions"))
    assert "missing key 'limit'" in error(lambda L, c: [L[i]["mlp"]["expert"].pop("limit") for i in (0, 5)])
    assert "must not be empty" in error(lambda L, c: c.update(width=0))
    # what may be left out
    cfg = copy.deepcopy(CONFIGS["odd"]())
    for k in ("logit_scale", "logit_softcap"):
        cfg.pop(k)
    cfg["layers"][3]["mixer"].pop("softcap")
    cfg["layers"][3]["mixer"]["mask"] = None
    cfg["layers"][3].pop("mlp")
    got = check("spec", written(tmp_path, cfg))
    assert got["logits"] == [1, 0] and got["layers"][3]["scores"][3:] == [0, 0] and got["layers"][3].get("poly") is None


def test_restatement_portions_equal_whole(tmp_path):
    for name in CONFIGS:
        cfg = CONFIGS[name]()
        m = pd.Model.load(write_folder(tmp_path / name, cfg, random_tensors(cfg, 5)))
        t = np.random.default_rng(2).integers(0, cfg["vocab"], size=23).tolist()
        s = m.sequence()
        whole = s.feed(t)
        u = m.sequence()
        parts = np.concatenate([u.feed(t[a:b]) for a, b in ((0, 1), (1, 3), (3, 20), (20, 23))])
        assert np.abs(whole - parts).max() < 1e-9 * np.abs(whole).max()
        assert np.allclose(s.margins, u.margins)


def test_recurrences_written_out():
    """Two tokens by hand: the bonus counts for the token itself only, what it writes is read by the next; a state space token reads what it writes."""
    r, k, v, w = (np.array(x, dtype=float).reshape(2, 1, -1) for x in ([[1, 2], [3, 4]], [[5, 6], [7, 8]], [[1], [10]], [[0.5, 0.25], [0.1, 0.1]]))
    o, S = pd.bonus_recurrence(r, k, v, w, np.array([[2.0, 3.0]]), np.zeros((1, 2, 1)))
    assert o.ravel().tolist() == [1 * 2 * 5 + 2 * 3 * 6, 3 * 5 + 4 * 6 + (3 * 2 * 7 + 4 * 3 * 8) * 10] and np.allclose(S.ravel(), [5 * 0.1 + 70, 6 * 0.1 + 80])
    y, S = pd.space_recurrence(v, k, r, np.array([[0.5], [2.0]]), np.array([[0.9], [0.25]]), np.array([3.0]), np.zeros((1, 2, 1)))
    assert np.allclose(y.ravel(), [0.5 * (5 + 12) + 3, 0.25 * 0.5 * (15 + 24) + 2 * (21 + 32) * 10 + 30])


def test_restatement_notices_planted_mistakes():
    """Each mistake, planted in the restatement, moves its logits far beyond what the device comparisons allow."""
    cfg = CONFIGS["odd"]()
    T = random_tensors(cfg, 3)
    t = np.random.default_rng(2).integers(0, cfg["vocab"], size=160).tolist()
    base = pd.Model(cfg, T).sequence().feed(t)

    def moved(change=lambda c, U: None, feed=None, **planted):
        c, U = copy.deepcopy(cfg), {k: np.copy(v) for k, v in T.items()}
        change(c, U)
        kept = {k: getattr(pd, k) for k in planted}
        try:
            for k, f in planted.items():
                setattr(pd, k, f)
            s = pd.Model(c, U).sequence()
            d = (feed(s) if feed else s.feed(t)) - base
        finally:
            for k, f in kept.items():
                setattr(pd, k, f)
        d -= d.mean(axis=1, keepdims=True)
        return np.sqrt((d * d).mean(axis=1)).max() / np.std(base)

    def lose(key, layers=None):
        def feed(s):
            a = s.feed(t[:70])
            for i, st in enumerate(s.state):
                if key in st and (layers is None or i in layers):
                    st[key] = np.zeros_like(st[key])
            return np.concatenate([a, s.feed(t[70:])])
        return feed

    def mixers(kind, **kw):
        def change(c, U):
            for l in c["layers"]:
                if l["type"] == kind:
                    l["mixer"].update({k: f(l["mixer"][k]) for k, f in kw.items()})
        return change

    def tensors(end, f):
        return lambda c, U: U.update({k: f(v) for k, v in T.items() if k.endswith(end)})
    seen, attend, space, mix, conv, group, route = pd.seen, pd.attend_head, pd.space_recurrence, pd.token_mix, pd.short_convolution, pd.gated_group_norm, pd.route

    def writes_first(r, k, v, w, u, S):
        o = np.zeros(v.shape)
        for i in range(len(r)):
            S = w[i][:, :, None] * S + k[i][:, :, None] * v[i][:, None, :]
            o[i] = np.einsum("hdv,hd->hv", S, r[i])
        return o, S

    def weighted_outputs(h, T, p, m):
        chosen, weight = pd.route(h, T[p + "router"], m["router"]["top"])
        out = np.zeros_like(h)
        for i, (c, w) in enumerate(zip(chosen, weight)):
            out[i] = sum(wj * pd.expert(h[i:i + 1], T, f"{p}e{j}.", m["expert"]["limit"])[0] for j, wj in zip(c, w))
        return out

    def renormalized(h, w, top):
        c, s = route(h, w, top)
        return c, s / s.sum(axis=1, keepdims=True)
    mistakes = dict(
        space_state=dict(feed=lose("S", (0, 5, 9, 10))), mixing_state=dict(feed=lose("S", (1, 4, 6, 8))), shared_layers_state=dict(feed=lose("S", (4, 5, 8))), previous_row=dict(feed=lose("h")),
        convolution_state=dict(feed=lose("conv")), lost_keys=dict(feed=lose("k")),
        window_in=dict(seen=lambda i, j, w: seen(i, j, w - 1)), window_out=dict(seen=lambda i, j, w: seen(i, j, w + 1)),
        sink=dict(attend_head=lambda *a: attend(*a[:-1], -1e9)), capped_sink=dict(attend_head=lambda *a: attend(*a[:-1], a[5] * np.tanh(a[-1] / a[5]))),
        no_cap=dict(attend_head=lambda q, k, v, p, s, c, *r: attend(q, k, v, p, s, None, *r)), cap=dict(change=mixers("attention", softcap=lambda v: v * 1.1)),
        scale=dict(change=mixers("attention", scale=lambda v: v * 1.1)), no_slope=dict(slope=lambda h, n: 0.0), next_slope=dict(slope=lambda h, n: 2.0 ** (-8.0 * h / n)),
        key_bias_only=dict(attend_head=lambda q, k, v, p, s, c, f, w, x: attend(q, k, v, p, s, c, f, w, x + f * np.mean(p))),
        write_first=dict(bonus_recurrence=writes_first), bonus=dict(change=tensors("mix.u", lambda v: v * 0)), mixes_swapped=dict(token_mix=lambda h, b, mu: mix(b, h, mu)),
        decay_weight=dict(channel_decay=lambda z: np.exp(-np.exp(z) * 1.1)), w0=dict(change=tensors("w0", lambda v: v + 0.2)),
        skip=dict(change=tensors("mix.D", lambda v: v * 0)), step=dict(space_recurrence=lambda x, B, C, dt, d, D, S: space(x, B, C, dt * 0 + 1, d, D, S)),
        step_bias=dict(change=tensors("dt_bias", lambda v: v + 0.2)), swapped=dict(space_recurrence=lambda x, B, C, *r: space(x, C, B, *r)),
        taps_reversed=dict(short_convolution=lambda u, b, w: conv(u, b, w[:, ::-1])), conv_bias=dict(change=tensors("conv.b", lambda v: v * 0)),
        norm_first=dict(gated_group_norm=lambda y, z, g, w, e: pd.root_norm(y.reshape(len(y), g, -1), e).reshape(y.shape) * w * pd.silu(z)),
        norm_groups=dict(gated_group_norm=lambda y, z, g, w, e: group(y, z, 1, w, e)),
        powers=dict(poly_norm=lambda z, a, e: a[0] * pd.root_norm(z, e) + a[1] * pd.root_norm(z, e) ** 2 + a[2] * pd.root_norm(z, e) ** 3 + a[3]),
        constant=dict(change=tensors("act", lambda v: v * [1, 1, 1, 0])), limit=dict(change=lambda c, U: [l["mlp"]["expert"].update(limit=9.0) for l in c["layers"] if l["mlp"] and "expert" in l["mlp"]]),
        gate_limited_below=dict(limited_gate=lambda g, u, m: (lambda a, b: a * pd.sigmoid(1.702 * a) * (b + 1))(np.clip(g, -m, m), np.clip(u, -m, m))),
        plain_silu=dict(limited_gate=lambda g, u, m: (lambda a, b: a * pd.sigmoid(a) * (b + 1))(np.minimum(g, m), np.clip(u, -m, m))),
        weighted_outputs=dict(routed_mlp=weighted_outputs), renormalized=dict(route=renormalized), positions=dict(change=lambda c, U: U.update(pos=np.roll(T["pos"], 1, axis=0))),
        logit_scale=dict(change=lambda c, U: c.update(logit_scale=0.75)), logit_cap=dict(change=lambda c, U: c.update(logit_softcap=None)),
        eps=dict(change=lambda c, U: c["norm"].update(eps=0.0)), own_cache=dict(feed=lambda s: (s.state.__setitem__(7, s.state[2]), s.feed(t))[1]))
    got = {name: moved(**m) for name, m in mistakes.items()}
    assert min(got.values()) > 2e-3, sorted(got.items(), key=lambda x: x[1])[:5]           # a hundred times the 32-bit limit
    assert moved() == 0
