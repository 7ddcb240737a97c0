"""The Natatar design without a device: its reader (through tests/layered_host_check.cpp) and the plain restatement against itself."""
import copy

import numpy as np
import pytest

from natatar_common import CONFIGS, random_config, random_tensors, sd, write_folder
from oracle.latent_decoder import rotation
from test_layered_host import check, written  # noqa: F401  (check is a fixture)


def near(a, b):
    return abs(a - b) <= 1e-6 * abs(b)


@pytest.mark.parametrize("name", list(CONFIGS) + [0, 1, 2])
def test_the_design_is_read_from_its_configuration(check, tmp_path, name):  # noqa: F811
    cfg = random_config(name) if isinstance(name, int) else CONFIGS[name]()
    got = check("spec", written(tmp_path, cfg))
    assert (got["architecture"], got["vocab"], got["width"], got["streams"]) == ("Natatar", cfg["vocab"], cfg["width"], cfg["streams"])
    assert got["tied_head"] and got["around_zero"] and got["positions"] == 0 and got["bigram"] == -1
    for key, want in (("eps", cfg["norm"]["eps"]), ("embedding_scale", cfg["embedding"]["scale"]), ("residual_mult", cfg["residual_mult"])):
        assert near(got[key], want)
    assert len(got["layers"]) == len(cfg["layers"])
    for g, l in zip(got["layers"], cfg["layers"]):
        m = l["mixer"]

        def heads(a, b, flags):
            assert a["sizes"] == [b[k] for k in ("heads", "kv_heads", "dim", "vdim")] and near(a["scale"], b["scale"]) and a["flags"] == flags
        if l["type"] == "attention":
            heads(g, m, [1, 1, 0, int(m.get("v_mix", False))])
            assert "freq" not in g
        elif l["type"] == "parallel":
            heads(g["left"], m["left"], [0, 0, 1, 0])
            f, mag = rotation(m["left"]["rot"])
            assert g["left"]["rot_dims"] == m["left"]["rot"]["dims"] and np.allclose(g["left"]["freq"], f, rtol=1e-13) and near(g["left"]["magnitude"], mag)
            assert g["right"][:3] == [m["right"][k] for k in ("heads", "dim", "vdim")] and near(g["right"][3], m["right"]["gate_cap"])
            assert near(g["factors"][0], m["left_scale"]) and near(g["factors"][1], m["right_scale"])
        else:
            assert g["sizes"] == [m[k] for k in ("heads", "kv_heads", "dim", "vdim", "conv")]
        assert g["ff"] == 0 and ("experts" in g) == bool(l["mlp"])
        if l["mlp"]:
            r = l["mlp"]["router"]
            assert g["experts"] == [r["experts"], 0, r["top"], l["mlp"]["expert"]["ff"]] and not g["correction"] and near(g["router_scale"], r.get("scale", 1.0))
            assert g["groups"] == [r["groups"][k] for k in ("count", "keep")] if "groups" in r else g["groups"] == [1, 1]


def test_bad_configurations_are_refused(check, tmp_path):  # noqa: F811
    def error(change):
        cfg = copy.deepcopy(CONFIGS["odd"]())
        change(cfg["layers"], cfg)
        return check("spec", written(tmp_path, cfg)).get("error", "")
    assert error(lambda L, c: None) == ""
    assert "unknown mixer" in error(lambda L, c: L[0].update(type="lightning"))
    assert "unknown feed-forward" in error(lambda L, c: L[0]["mlp"].update(kind="dense"))
    for i, key in ((0, "vdim"), (1, "dim"), (1, "conv")):
        assert "size is zero" in error(lambda L, c: L[i]["mixer"].update({key: 0}))
    assert "size is zero" in error(lambda L, c: L[2]["mixer"]["left"].update(dim=0))
    assert "size is zero" in error(lambda L, c: L[2]["mixer"]["right"].update(heads=0))
    assert "size is zero" in error(lambda L, c: L[0]["mlp"]["expert"].update(ff=0))
    assert "multiple of kv_heads" in error(lambda L, c: L[0]["mixer"].update(heads=5))
    assert "multiple of kv_heads" in error(lambda L, c: L[1]["mixer"].update(kv_heads=4))
    assert "scale is zero" in error(lambda L, c: L[0]["mixer"].update(scale=0))
    assert "rot.dims" in error(lambda L, c: L[2]["mixer"]["left"]["rot"].update(dims=22))
    assert "rot.dims" in error(lambda L, c: L[2]["mixer"]["left"]["rot"].update(dims=9))
    assert "gate_cap" in error(lambda L, c: L[2]["mixer"]["right"].update(gate_cap=0))
    assert "value columns" in error(lambda L, c: L[4]["mixer"].update(vdim=13))
    assert "not true or false" in error(lambda L, c: L[4]["mixer"].update(v_mix=3))
    assert "multiple of groups.count" in error(lambda L, c: L[0]["mlp"]["router"]["groups"].update(count=4))
    assert "groups.keep" in error(lambda L, c: L[0]["mlp"]["router"]["groups"].update(keep=4))
    assert "router.top" in error(lambda L, c: L[0]["mlp"]["router"].update(top=5))
    assert "missing key 'streams'" in error(lambda L, c: c.pop("streams"))
    assert "must not be empty" in error(lambda L, c: c.update(streams=0))
    # what may be left out
    cfg = copy.deepcopy(CONFIGS["odd"]())
    for k in ("embedding", "residual_mult"):
        cfg.pop(k)
    for k in ("groups", "scale"):
        cfg["layers"][0]["mlp"]["router"].pop(k)
    got = check("spec", written(tmp_path, cfg))
    assert (got["embedding_scale"], got["residual_mult"], got["layers"][0]["groups"], got["layers"][0]["router_scale"]) == (1, 1, [1, 1], 1)


def test_ranks_come_from_the_tensors(check, tmp_path):  # noqa: F811
    cfg = CONFIGS["odd"]()
    T = random_tensors(cfg, 1)
    f = write_folder(tmp_path, cfg, T) + "/model.safetensors"
    assert check("rows", f, "l1.mix.a1") == len(T["l1.mix.a1"]) and check("rows", f, "l1.mix.g1") == len(T["l1.mix.g1"])
    assert "no tensor named" in check("rows", f, "l1.mix.a3")["error"] and "no rows" in check("rows", f, "l3.mix.vmix")["error"]


def test_restatement_portions_equal_whole(tmp_path):
    for name in CONFIGS:
        cfg = CONFIGS[name]()
        m = sd.Model.load(write_folder(tmp_path / name, cfg, random_tensors(cfg, 5)))
        t = np.random.default_rng(2).integers(0, cfg["vocab"], size=23).tolist()
        s = m.sequence()
        whole = s.feed(t)
        u = m.sequence()
        parts = np.concatenate([u.feed(t[a:b]) for a, b in ((0, 1), (1, 3), (3, 20), (20, 23))])
        assert np.abs(whole - parts).max() < 1e-9 * np.abs(whole).max()
        assert np.allclose(s.margins, u.margins)


def test_choice_within_groups_and_its_margin():
    z = np.array([[5.0, 0.0, 4.0, 3.9, 4.5, -9.0]])
    r = dict(top=3, scale=2.0, groups=dict(count=3, keep=2))
    chosen, w = sd.route(z, np.eye(6), r)
    s = np.exp(z) / np.exp(z).sum()
    assert chosen.tolist() == [[0, 4, 1]] and np.allclose(w, 2.0 * s[0, [0, 4, 1]])      # the second group's 4.0 and 3.9 are left out
    assert np.isclose(sd.choice_margin(z, np.eye(6), r)[0], 0.5)                         # its best against the third's
    assert np.isclose(sd.choice_margin(z, np.eye(6), dict(r, top=2))[0], 0.5) and np.isclose(sd.choice_margin(z, np.eye(6), dict(top=3))[0], 0.1)
    assert np.isinf(sd.choice_margin(z, np.eye(6), dict(top=6))).all()


def test_restatement_notices_planted_mistakes():
    """Each mistake, planted in the restatement, moves its logits far beyond what the device comparisons allow."""
    cfg = CONFIGS["odd"]()
    T = random_tensors(cfg, 3)
    t = np.random.default_rng(2).integers(0, cfg["vocab"], size=90).tolist()
    base = sd.Model(cfg, T).sequence().feed(t)

    def moved(change=lambda c, U: None, feed=None, **planted):
        c, U = copy.deepcopy(cfg), {k: np.copy(v) for k, v in T.items()}
        change(c, U)
        kept = {k: getattr(sd, k) for k in planted}
        try:
            for k, f in planted.items():
                setattr(sd, k, f)
            s = sd.Model(c, U).sequence()
            d = (feed(s) if feed else s.feed(t)) - base
        finally:
            for k, f in kept.items():
                setattr(sd, k, f)
        d -= d.mean(axis=1, keepdims=True)
        return np.sqrt((d * d).mean(axis=1)).max() / np.std(base)

    def lose(key, side=None):
        def feed(s):
            a = s.feed(t[:40])
            for st in s.state:
                st = st[side] if side else st
                for k in list(st):
                    if k.endswith(key):
                        st[k] = np.zeros_like(st[k])
            return np.concatenate([a, s.feed(t[40:])])
        return feed

    def mixers(kind, side=None, **kw):
        def change(c, U):
            for l in c["layers"]:
                if l["type"] == kind:
                    m = l["mixer"][side] if side else l["mixer"]
                    m.update({k: f(m[k]) for k, f in kw.items() if k in m})
        return change

    def tensors(end, f):
        return lambda c, U: U.update({k: f(v) for k, v in T.items() if k.endswith(end)})

    def routers(**kw):
        return lambda c, U: [l["mlp"]["router"].update({k: v for k, v in kw.items() if k in l["mlp"]["router"]}) for l in c["layers"] if l["mlp"]]

    def one_head_at_a_time(x, w, eps):          # norms per head of 10 instead of over a projection
        y = x.reshape(len(x), -1, 10) if x.ndim == 2 and x.shape[1] in (90, 30) and len(w) in (90, 30) else None
        return rms(x, w, eps) if y is None else (y / np.sqrt((y * y).mean(axis=-1, keepdims=True) + eps)).reshape(x.shape) * w

    def reads_before_writing(q, k, v, g, beta, S):
        o = np.zeros(v.shape)
        for i in range(len(q)):
            S = g[i][:, :, None] * S
            o[i] = np.einsum("hdv,hd->hv", S, q[i])
            S = S + k[i][:, :, None] * (beta[i][:, None] * (v[i] - np.einsum("hdv,hd->hv", S, k[i])))[:, None, :]
        return o, S
    rms, attend, conv, write, unit, allowed, rotate = (sd.rms_norm, sd.softmax_attend, sd.short_convolution, sd.write_streams, sd.unit, sd.allowed_experts, sd.rotate)
    mistakes = dict(
        delta_state=dict(feed=lose("S")), memory_state=dict(feed=lose("S", "right")), memory_normalizer=dict(feed=lose("n", "right")),
        memory_maximum=dict(feed=lose("m", "right")), convolution_state=dict(feed=lose(".q")), value_convolution_state=dict(feed=lose("mix.v")),
        scale=dict(change=mixers("attention", scale=lambda v: v * 1.1)), left_scale=dict(change=mixers("parallel", "left", scale=lambda v: v * 1.1)),
        factors=dict(change=mixers("parallel", left_scale=lambda v: v * 1.05)), cap=dict(change=mixers("parallel", "right", gate_cap=lambda v: v * 1.3)),
        key_biases=dict(change=tensors("k.b", lambda v: v * 0)), value_biases=dict(change=tensors("v.b", lambda v: v * 0)),
        values_unmixed=dict(change=mixers("attention", v_mix=lambda v: False)), values_of_one_layer_unmixed=dict(change=lambda c, U: U.update({"l4.mix.vmix": np.float32(0)})),
        norm_per_head=dict(rms_norm=one_head_at_a_time), one_key_late=dict(softmax_attend=lambda q, k, v, s, p: attend(q, k, v, s, np.maximum(np.asarray(p) - 1, 0))),
        angles=dict(rotate=lambda x, p, rot: rotate(x, p, dict(rot, scaling=None))), other_pairs=dict(rotate=lambda x, p, rot: rotate(x[..., ::-1], p, rot)[..., ::-1]),
        taps_reversed=dict(short_convolution=lambda u, b, w: conv(u, b, w[:, ::-1])), read_before_write=dict(delta_recurrence=reads_before_writing),
        not_unit=dict(unit=lambda x: unit(x) * 1.1),
        mix_transposed=dict(write_streams=lambda X, m, o, y, f: write(X, m.T, o, y, f)),
        one_stream_after_the_other=dict(write_streams=lambda X, m, o, y, f: np.stack([(z := write(X, m, o, y, f))[0], *write(np.concatenate([z[:1], X[1:]]), m, o, y, f)[1:]])),
        shares=dict(change=tensors(".out", lambda v: v * 0 + 1)), residual=dict(change=lambda c, U: c.update(residual_mult=1.0)),
        embedding=dict(change=lambda c, U: c["embedding"].update(scale=1.0)), eps=dict(change=lambda c, U: c["norm"].update(eps=0.0)),
        plain_norms=dict(around_zero_norm=lambda x, w, eps: rms(x, w, eps)), groups=dict(allowed_experts=lambda s, c, k: allowed(s, 1, 1)),
        router_scale=dict(change=routers(scale=1.0)), decay_bias=dict(change=tensors("dt_bias", lambda v: v + 3)), gate_bias=dict(change=tensors("f.b", lambda v: v + 0.1)))
    got = {name: moved(**m) for name, m in mistakes.items()}
    assert min(got.values()) > 2e-3, sorted(got.items(), key=lambda x: x[1])[:5]           # a hundred times the 32-bit limit
    assert moved() == 0
