"""The Fomunex design through the framework's model folders, step function, paged cache, state slots and scheduler, against the plain
restatement in oracle/prenorm_decoder.py: whole prompts, portions, single tokens, mixed batches, pages and slots used again, keys at the edges of
windows and pages."""
import importlib
import json
import os
import subprocess

import numpy as np
import pytest

pytestmark = pytest.mark.gpu

from fomunex_common import CONFIGS, attention, dense, make_folder, model, pd, random_config, random_tensors, write_folder  # noqa: E402
from pimosun_common import layered, logits_error, m40  # noqa: E402
from test_gpu_gulidra import assert_close, assert_logits  # noqa: E402

sch = importlib.import_module("m40-llm_amd.scheduler")
DTYPES = ["float32", "bfloat16"]
# (dtype, form of the portions' attention: 0 the cheaper, 1 that of single tokens, 2 that of long portions)
FORMS = [("float32", 0), ("bfloat16", 1), ("bfloat16", 2)]


@pytest.fixture(scope="module")
def ctx():
    yield m40.Context(0)


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    made = {}

    def get(name):
        if name not in made:
            made[name] = make_folder(tmp_path_factory.mktemp("fomunex_" + name), name)
        return made[name]
    return get


@pytest.fixture(scope="module")
def expected(folders):
    """(tokens, logits [tokens][vocab], residuals [layers][tokens][width], margins of the experts' choice) of a sequence of n tokens,
    computed whole."""
    kept, models = {}, {}

    def get(name, n, seed=0):
        if (name, n, seed) not in kept:
            m = models.setdefault(name, pd.Model.load(folders(name)))
            t = np.random.default_rng(1000 * seed + n).integers(0, m.cfg["vocab"], size=n)
            s = m.sequence()
            kept[name, n, seed] = (t, s.feed(t.tolist()), np.stack(s.layer_outputs), np.array(s.margins))
        return kept[name, n, seed]
    return get


def open_model(ctx, folder, dtype, max_tokens=1024, slots=4, **kw):
    return layered.LayeredModel.open(ctx, folder, dtype, max_tokens, slots, **kw)


@pytest.mark.parametrize("dtype,form", FORMS)
@pytest.mark.parametrize("name,n", [("odd", 150), ("even", 200), ("wide", 140), ("one", 70)])
def test_residual_after_every_layer_and_logits_of_a_whole_prompt(ctx, folders, expected, name, n, dtype, form):
    t, want, res, margins = expected(name, n)
    m = open_model(ctx, folders(name), dtype, portion_form=form)
    x = m.step_layers(0, t, *[res.shape[i] for i in (0, 2)])
    for i in range(len(res)):
        e = np.sqrt(((x[i] - res[i]) ** 2).mean(axis=-1)) / np.sqrt((res[i] ** 2).mean())
        assert_close(e, dtype, margins, i)
    m.release(0)
    assert_logits(m.step([(1, t, range(n))]), want, dtype, margins)
    m.close()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name,n,first", [("odd", 135, 60), ("even", 200, 1), ("wide", 90, 66), ("one", 70, 62)])
def test_token_by_token_equals_the_whole_prompt(ctx, folders, expected, name, n, first, dtype):
    t, want, _, margins = expected(name, n)
    m = open_model(ctx, folders(name), dtype)
    got = [m.step([(2, t[:first], range(first))])]
    for i in range(first, n):
        got.append(m.step([(2, t[i:i + 1], [0])]))
    assert_logits(np.concatenate(got), want, dtype, margins)
    m.close()


@pytest.mark.parametrize("dtype,form", FORMS + [("bfloat16", 0)])
@pytest.mark.parametrize("name,n", [("odd", 330), ("even", 330), ("wide", 200)])
@pytest.mark.parametrize("cut", [[2], [3, 2, 61, 64, 66], [63, 1], [128, 5], [65], [200, 2]])
def test_portions_of_any_size(ctx, folders, expected, name, n, cut, dtype, form):
    t, want, _, margins = expected(name, n)
    m = open_model(ctx, folders(name), dtype, portion_form=form)
    at, k, got = 0, 0, []
    while at < n:
        c = min(cut[k % len(cut)], n - at)
        got.append(m.step([(0, t[at:at + c], range(c))]))
        at, k = at + c, k + 1
    assert_logits(np.concatenate(got), want, dtype, margins, cut)
    m.close()


@pytest.mark.parametrize("dtype,form", FORMS + [("bfloat16", 0)])
@pytest.mark.parametrize("max_rows", [0, 7, 100])
def test_mixed_batches_with_pages_and_slots_used_again(ctx, folders, expected, dtype, form, max_rows):
    """Twelve sequences through four slots and a pool that holds four of them: portions of some beside single tokens of others,
    sequences left out for a step, every position compared; then the pool is whole again."""
    rng = np.random.default_rng(17)
    lens = [5, 64, 65, 150, 127, 2, 129, 70, 1, 192, 128, 33]
    m = open_model(ctx, folders("odd"), dtype, max_tokens=4 * 192, max_rows=max_rows, portion_form=form)
    free0 = m.free_pages()
    waiting, live, free, errors, margins = list(range(len(lens))), {}, [0, 1, 2, 3], [], []
    seqs = {i: expected("odd", n, seed=1 + i) for i, n in enumerate(lens)}
    spread = np.std(np.concatenate([s[1] for s in seqs.values()]))
    while waiting or live:
        while waiting and free:
            live[waiting.pop(0)] = [free.pop(rng.integers(len(free))), 0]
        entries, rows = [], []
        for i in rng.permutation(list(live)):
            if len(live) > 1 and rng.random() < 0.2:
                continue
            slot, at = live[i]
            t = seqs[i][0]
            c = 1 if at > 0 and rng.random() < 0.5 else int(rng.integers(1, 90))
            c = min(c, len(t) - at)
            entries.append((slot, t[at:at + c], range(c)))
            rows += [(i, at + k) for k in range(c)]
            live[i][1] = at + c
        if not entries:
            continue
        got = m.step(entries)
        want = np.stack([seqs[i][1][p] for i, p in rows])
        e = logits_error(got, want) * np.std(want) / spread
        if dtype == "float32":
            assert_close(e, dtype, None, (rows[0], len(entries)))
        errors.append(e)
        margins += [seqs[i][3][p] for i, p in rows]
        for i in [i for i, (slot, at) in live.items() if at == lens[i]]:
            slot, _ = live.pop(i)
            m.release(slot)
            free.append(slot)
    assert_close(np.concatenate(errors), dtype, margins)
    assert m.free_pages() == free0
    m.close()


@pytest.mark.parametrize("seed", range(24))
def test_random_configurations(ctx, tmp_path, seed):
    """Layers of any kind and size in any order: portions, two sequences at a time, single tokens."""
    cfg = random_config(seed)
    folder = write_folder(tmp_path, cfg, random_tensors(cfg, seed))
    mod = pd.Model.load(folder)
    toks = [np.random.default_rng(seed + k).integers(0, cfg["vocab"], size=140) for k in (0, 50)]
    seqs = [mod.sequence() for _ in toks]
    want = np.stack([s.feed(t.tolist()) for s, t in zip(seqs, toks)])
    margins = np.array([s.margins for s in seqs])
    for dtype in DTYPES:
        m = open_model(ctx, folder, dtype, max_tokens=384, slots=2)
        at, got = [0, 0], [[], []]
        for cuts in ((70, 3), (1, 65), (34, 2), (1, 1), (1, 40), (1, 1), (30, 1), (2, 27)):
            out = m.step([(k, toks[k][at[k]:at[k] + c], range(c)) for k, c in enumerate(cuts)])
            got[0].append(out[:cuts[0]]); got[1].append(out[cuts[0]:])
            at = [a + c for a, c in zip(at, cuts)]
        assert at == [140, 140]
        e = np.concatenate([logits_error(np.concatenate(got[k]), want[k]) for k in (0, 1)])
        assert_close(e, dtype, margins.reshape(-1), seed, factor=2)
        m.close()


@pytest.mark.parametrize("dtype,form", FORMS)
def test_batch_of_unequal_requests_equals_each_alone(ctx, folders, expected, dtype, form):
    m = open_model(ctx, folders("even"), dtype, max_tokens=1024, portion_form=form)
    lens = [200, 3, 129, 64]
    seqs = [expected("even", n, seed=40) for n in lens]
    alone = []
    for t, _, _, _ in seqs:
        alone.append(m.step([(0, t, range(len(t)))]))
        m.release(0)
    together = m.step([(i, t, range(len(t))) for i, (t, _, _, _) in enumerate(seqs)])
    at = 0
    for (t, want, _, margins), a in zip(seqs, alone):
        b = together[at:at + len(t)]
        assert_logits(b, want, dtype, margins)
        assert_close(logits_error(a, b.astype(np.float64)), dtype, margins, factor={"float32": 0.25, "bfloat16": 0.7}[dtype])
        at += len(t)
    m.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_first_tokens_of_a_sequence_on_used_slots(ctx, folders, dtype):
    """States and convolutions start at zero whatever ran in the slot before; a cut inside the convolution's reach changes nothing."""
    mod = pd.Model.load(folders("odd"))
    m = open_model(ctx, folders("odd"), dtype)
    m.step([(1, np.arange(60) % 101, [])])
    m.release(1)
    for first, cut in (([7], 1), ([0, 0, 5, 9, 9, 100], 1), ([100, 3, 100, 4, 8], 2), ([1, 2, 3, 4, 5, 6, 7], 3)):
        s = mod.sequence()
        want = s.feed(first)
        got = [m.step([(1, first[i:i + cut], range(len(first[i:i + cut])))]) for i in range(0, len(first), cut)]
        assert_logits(np.concatenate(got), want, dtype, s.margins, (first, cut))
        m.release(1)
    m.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_wanted_places_any_order_and_none(ctx, folders, expected, dtype):
    t, want, _, margins = expected("odd", 135)
    m = open_model(ctx, folders("odd"), dtype)
    assert m.step([(0, t[:40], [])]).shape == (0, want.shape[1])
    got = m.step([(0, t[40:], [94, 0, 3, 3])])
    assert_logits(got, want[[134, 40, 43, 43]], dtype, margins[[134, 40, 43, 43]])
    m.close()


def test_bad_steps_are_refused_and_change_nothing(ctx, folders, expected):
    t, want, _, margins = expected("odd", 135)
    m = open_model(ctx, folders("odd"), "float32", max_tokens=192, slots=2)
    m.step([(0, t[:64], [])])
    for bad in ([(0, [5000], [])], [(2, [1], [])], [(0, [1], [1])], [(0, [1], []), (0, [2], [])], [(0, [], [])],
                [(1, list(range(100)) + [0] * 40, [])]):
        with pytest.raises(RuntimeError):
            m.step(bad)
    m.release(1)
    assert m.length(0) == 64
    assert_logits(m.step([(0, t[64:], range(71))]), want[64:], "float32")
    m.close()


@pytest.mark.parametrize("dtype,mode,guard", [("float32", 0, None), ("float32", 2, None), ("bfloat16", 2, None), ("float32", 2, 1e9)])
def test_long_greedy_decoding_equals_the_oracle(ctx, folders, dtype, mode, guard):
    """The device-driven loop (plain launches and replayed from a graph) over several page borders; a huge tie guard sends every run through
    the host sampler, which starts again from the states before the loop."""
    mod = pd.Model.load(folders("odd"))
    m = open_model(ctx, folders("odd"), dtype)
    m.set_mode(mode)
    if guard:
        m.set_tie_guard(guard)
    prompt = np.random.default_rng(5).integers(0, 101, size=50).tolist()
    ids, gaps = m.decode_greedy(0, prompt, 160)
    assert m.last_timed_host_fallback() == bool(guard)
    s = mod.sequence()
    want = s.feed(ids[:-1].tolist())[len(prompt) - 1:]
    pick = ids[len(prompt):]
    if dtype == "float32":
        assert np.array_equal(want.argmax(axis=1), pick)
    behind = (want.max(axis=1) - want[np.arange(len(pick)), pick]) / np.std(want)
    assert np.sort(behind)[int(0.97 * len(behind))] <= 4 * {"float32": 1e-4, "bfloat16": 0.03}[dtype] and behind.max() < 1.0
    assert m.length(0) == len(prompt) + 159
    # the loop's state carries on: the next token continues behind it
    got = m.step([(0, ids[-1:], [0])])
    assert_logits(got, s.feed(ids[-1:].tolist()), dtype, s.margins[-1:], factor=2)
    m.close()


def test_greedy_batch_loop_on_any_slots_equals_single_sequences(ctx, folders):
    m = open_model(ctx, folders("odd"), "float32")
    rng = np.random.default_rng(6)
    prompts = [rng.integers(0, 101, size=n).tolist() for n in (3, 63, 90)]
    alone = []
    for p in prompts:
        ids, _ = m.decode_greedy(1, p, 40)
        alone.append(ids[len(p):])
        m.release(1)
    slots = [3, 0, 2]
    last = m.step([(s, p, [len(p) - 1]) for s, p in zip(slots, prompts)]).argmax(axis=1)
    ids, _ = m.decode_batch_timed(slots, [len(p) for p in prompts], last, 5, 34)
    for a, f, b in zip(alone, last, ids):
        assert a.tolist() == [int(f)] + b.tolist()
    m.close()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("max_rows,max_tokens", [(0, 1024), (24, 320)])
def test_scheduler_serves_requests_as_each_alone(ctx, folders, dtype, max_rows, max_tokens):
    """Arrivals over time, prompts cut by the tick's row limit, requests that wait for pages: every request generates (32-bit) what the
    oracle picks for it alone."""
    m = open_model(ctx, folders("odd"), dtype, max_tokens=max_tokens, slots=3, max_rows=max_rows)
    mod = pd.Model.load(folders("odd"))
    rng = np.random.default_rng(9)
    specs = [(rng.integers(0, 101, size=n).tolist(), g) for n, g in ((9, 20), (130, 12), (64, 3), (1, 30), (77, 9), (40, 40))]
    s = sch.Scheduler.for_model(m)
    free0, rids, pending, ticks, mixed = m.free_pages(), {}, list(enumerate(specs)), 0, 0
    while pending or s.active():
        while pending and s.available_slots() and (ticks == 0 or ticks % 3 == 0):
            i, (p, g) = pending.pop(0)
            rids[i] = s.submit(p, max_tokens=g)
        rep = s.tick()
        mixed += bool(rep.prefill_rows and rep.decode_rows)
        ticks += 1
        assert ticks < 400
    assert mixed > 0 and m.free_pages() == free0
    behind = []
    for i, (p, g) in enumerate(specs):
        assert s.state(rids[i]) == "complete", s.error(rids[i])
        got = s.generated(rids[i])
        assert len(got) == g
        want = mod.sequence().feed((p + got)[:-1])[len(p) - 1:]
        if dtype == "float32":
            assert want.argmax(axis=1).tolist() == got, i
        behind += ((want.max(axis=1) - want[np.arange(g), got]) / np.std(want)).tolist()
    assert np.sort(behind)[int(0.97 * len(behind))] <= 4 * {"float32": 1e-4, "bfloat16": 0.03}[dtype] and max(behind) < 1.0
    s.close()
    m.close()


def test_command_line_generates_what_the_oracle_picks(ctx, folders, capsys):
    gen = importlib.import_module("m40-llm_amd.generate")
    mod = pd.Model.load(folders("odd"))
    prompts = [[3, 1, 4, 1, 5], [9] * 70, [2]]
    gen.main(["--model", folders("odd"), "--dtype", "float32", "--max-tokens", "9", "--slots", "2"] + sum((["--prompt", ",".join(map(str, p))] for p in prompts), []))
    lines = [json.loads(x) for x in capsys.readouterr().out.splitlines()]
    assert [x["prompt"] for x in lines] == prompts
    for x in lines:
        want = mod.sequence().feed((x["prompt"] + x["generated"])[:-1])[len(x["prompt"]) - 1:]
        assert want.argmax(axis=1).tolist() == x["generated"]


def test_trace_replay(ctx, folders, expected, tmp_path):
    """bin/trace_run over a small trace in 32-bit: requests cut into steps, ended and admitted on slots that were used before."""
    t, want, _, margins = expected("odd", 135)
    V = want.shape[1]
    steps, rows = [], []

    def step(entries, end=()):
        steps.append(json.dumps({"step": len(steps), "entries": [{"id": i, "tokens": t[a:b].tolist(), "want": w} for i, a, b, w in entries], "end": list(end)}))
        rows.append([a + x for _, a, _, w in entries for x in w])
    step([("a", 0, 70, [69, 3])])
    step([("b", 0, 2, []), ("a", 70, 71, [])])
    step([("b", 2, 100, [0, 97]), ("a", 71, 72, [0]), ("c", 0, 1, [0]), ("d", 0, 5, [4])], ["a", "c"])
    step([("e", 0, 64, [63]), ("b", 100, 135, [34])], ["b"])
    step([("e", 64, 66, [0, 1])], ["e"])
    exe = os.path.join(m40.ROOT, "bin", "trace_run")
    p = subprocess.run([exe, "--model", folders("odd"), "--dtype", "float32", "--out", str(tmp_path), "--max-tokens", str(4 * 192)], input="\n".join(steps) + "\n",
                       capture_output=True, text=True, timeout=100)
    assert p.returncode == 0, p.stderr[-2000:]
    assert p.stdout.split("\n")[:-1] == ["done %d" % i for i in range(5)]
    for i, r in enumerate(rows):
        f = tmp_path / f"{i}.f32"
        if not r:
            assert not f.exists()
            continue
        assert_logits(np.fromfile(f, dtype="<f4").reshape(len(r), V), want[r], "float32")


def edge_model(tmp_path, window):
    """One attention layer in which token 1 is the only key that token 2 looks for: whether it is seen decides the logits."""
    cfg = model(24, 64, [(attention(4, 2, 16, 12, window, 30.0, scale=1.6), None)], positions=400, logit_softcap=40.0)
    T = random_tensors(cfg, 1)
    rng = np.random.default_rng(2)
    T["embed"] = np.zeros((24, 64), np.float32)
    T["embed"][np.arange(24), np.arange(24)] = 8.0             # a direction a token
    T["pos"] *= 0.0
    for c, token, heads in (("q", 2, 4), ("k", 1, 2)):
        w = np.zeros((heads * 16, 64), np.float32)
        w[:, :24] = rng.standard_normal((heads * 16, 24))
        w.reshape(heads, 16, 64)[:, :4] = 0.0
        w[:, token] = np.tile([1.0] * 4 + [0.0] * 12, heads)      # the only one with these dimensions
        T["l0.mix." + c] = w
    folder = write_folder(tmp_path / str(window), cfg, T)
    return folder, pd.Model.load(folder)


@pytest.mark.parametrize("dtype,form", FORMS + [("bfloat16", 0)])
@pytest.mark.parametrize("window", [1, 2, 31, 63, 64, 65, 100, 128, 130])
def test_key_just_inside_and_just_outside_the_window(ctx, tmp_path, window, dtype, form):
    folder, mod = edge_model(tmp_path, window)
    m = open_model(ctx, folder, dtype, portion_form=form)
    for at in (0, 5, 63, 64, 100):
        t = np.random.default_rng(at).integers(3, 24, size=at + window + 12)
        t[at] = 1
        near, far = at + window - 1, at + window                 # the last position that sees it, and the next
        if window > 1:
            t[near] = 2
        t[far] = 2
        want = mod.sequence().feed(t.tolist())
        if window > 1:
            d = want[near] - want[far]
            assert np.std(d) > 0.3 * np.std(want)
        for cut in ([len(t)], [near, 1, 1, 1], [max(near - 3, 1), 2, 2, 2], [1] * 40 if len(t) <= 40 else [40, 30]):
            got, done, k = [], 0, 0
            while done < len(t):
                c = min(cut[k % len(cut)] or 1, len(t) - done)
                got.append(m.step([(3, t[done:done + c], range(c))]))
                done, k = done + c, k + 1
            m.release(3)
            assert_logits(np.concatenate(got), want, dtype, None, (window, at, cut))
    m.close()


def test_no_more_tokens_than_positions(ctx, folders, tmp_path):
    cfg = CONFIGS["one"]()
    cfg["max_positions"] = 70
    m = open_model(ctx, write_folder(tmp_path, cfg, random_tensors(cfg, 1)), "float32")
    m.step([(0, [1] * 69, [])])
    with pytest.raises(RuntimeError):
        m.step([(0, [1, 2], [])])
    assert m.step([(0, [1], [0])]).shape == (1, cfg["vocab"])
    m.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_layers_that_share_tensors_equal_layers_that_have_copies(ctx, folders, tmp_path, dtype):
    cfg = CONFIGS["odd"]()
    T = random_tensors(cfg, 3)
    copies = json.loads(json.dumps(cfg))
    for i, l in enumerate(copies["layers"]):
        own = pd.tensors_of(cfg["layers"], i)
        l.pop("weights_of", None)
        T.update({f"l{i}." + k[len(f"l{own}."):]: v for k, v in list(T.items()) if k.startswith(f"l{own}.")})
    t = np.random.default_rng(0).integers(0, 101, size=90)
    out = []
    for folder in (folders("odd"), write_folder(tmp_path, copies, T)):
        m = open_model(ctx, folder, dtype)
        out.append(np.concatenate([m.step([(0, t[:70], range(70))]), m.step([(0, t[70:71], [0])]), m.step([(0, t[71:], range(19))])]))
        m.close()
    assert np.array_equal(*out)


def test_a_model_with_other_optional_parts(ctx, tmp_path):
    """No window, no cap on scores, none on logits, no scale."""
    cfg = model(60, 48, [(attention(4, 2, 24, 16, 5, 5.0), dense(40)), (attention(2, 1, 16, 16, 70, 3.0), None)])
    for k in ("logit_scale", "logit_softcap"):
        cfg.pop(k)
    m0 = cfg["layers"][0]["mixer"]
    m0.pop("softcap")
    m0["mask"] = None
    folder = write_folder(tmp_path, cfg, random_tensors(cfg, 4))
    t = np.random.default_rng(0).integers(0, 60, size=200)
    want = pd.Model.load(folder).sequence().feed(t.tolist())
    for dtype, form in FORMS:
        m = open_model(ctx, folder, dtype, portion_form=form)
        assert_logits(np.concatenate([m.step([(0, t[:150], range(150))])] + [m.step([(0, t[i:i + 1], [0])]) for i in range(150, 200)]), want, dtype)
        m.close()
