"""The building blocks of pre-norm layers one by one, through the C ABI: products whose columns read different parts of a row, experts weighted at
their input, attention with capped scores, slopes, windows and sinks, token mixes, the normed polynomial, gate and norm over parts of a row,
convolution with bias, time mixing and the stepped linear attention token by token and chunk by chunk.  Inputs are made so that one key out of
place, a window one token off, a sink left out, a lost state or a decay off by one token shows at once."""
import ctypes as C

import numpy as np
import pytest

pytestmark = pytest.mark.gpu

from fomunex_common import pd  # noqa: E402
from pimosun_common import as_act, c_struct, close_to, from_act, ld, m40, pack_tiles, unpack_tiles, up32  # noqa: E402
from test_gpu_layer_kernels import ACT, DTYPES, ROWS, act_type, bf16w, call, gemm, rounded  # noqa: E402
from test_gpu_stream_kernels import FORMS, PATHS, RUNS, Cache, run_recurrence, state_close  # noqa: E402
from test_gpu_sublayer_kernels import LONE, dev, filled, u32  # noqa: E402

Gemm, Update, Split, Attn, Route, Mix, Space, Light, Mixing = (c_struct("M40llm" + n) for n in ("PackedGemm", "StreamUpdate", "PairSplit", "PairAttention", "Route", "TokenMix",
                                                                                               "SpaceSplit", "Lightning", "TimeMixing"))
PROJECT, TANH, CAP = 5, 10, 11
LIMITED = 2


@pytest.fixture(scope="module")
def ctx():
    yield m40.Context(0)


# ---- products --------------------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows", ROWS)
@pytest.mark.parametrize("k,segments,last", [(64, 3, 40), (300, 2, 256), (40, 4, 16)])
def test_columns_that_read_their_own_part_of_a_row(ctx, dtype, rows, k, segments, last):
    """Segments of 256 columns, each from its own k columns of the row; the last one's go through tanh to the operand."""
    rng = np.random.default_rng(rows + k)
    pad = up32(k)
    A = np.zeros((rows, (segments + 1) * pad))
    W = np.zeros((segments * 256 + last, k), np.float32)
    want = []
    for s in range(segments + 1):
        n = 256 if s < segments else last
        A[:, s * pad:s * pad + k] = rng.standard_normal((rows, k))
        W[s * 256:s * 256 + n] = bf16w(rng, n, k)
        want.append(rounded(A[:, s * pad:s * pad + k], dtype) @ W[s * 256:s * 256 + n].T.astype(np.float64))
    dA, dW = ctx.to_device(pack_tiles(as_act(A, dtype))), ctx.to_device(pack_tiles(ld.f32_to_bf16(W)))
    lda, n_tiles = (segments + 1) * pad, segments * 16 + (last + 15) // 16
    plain, act = ctx.to_device(np.full((rows, segments * 256), 7.0, np.float32)), ctx.to_device(filled((rows + 15) // 16 * 16 * up32(last), dtype))
    g = Gemm(act_dtype=ACT[dtype], epilogue=TANH, a=dA.ptr, lda=lda, a_batch=pad, segment_tiles=16, w=dW.ptr, n_tiles=n_tiles, k_tiles=pad // 32, rows=rows, batches=1,
             plain_tiles=segments * 16, out_f32=plain.ptr, ld_out=segments * 256, out_act=act.ptr, ld_act=up32(last))
    call(ctx, "m40llm_ext_packed_gemm_async", C.byref(g), 1)
    got = plain.download(np.float32, (rows, segments * 256))
    for s in range(segments):
        close_to(got[:, s * 256:(s + 1) * 256], want[s], "float32", factor=2)
    close_to(from_act(unpack_tiles(act.download(act_type(dtype), ((rows + 15) // 16 * 16 * up32(last),)), rows, up32(last)), dtype)[:, :last], np.tanh(want[-1]), dtype, factor=2)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows", [1, 70, 200])
@pytest.mark.parametrize("scale,cap", [(0.25, 3.0), (2.0, 0.0), (1.0, 1e4)])
def test_capped_columns(ctx, dtype, rows, scale, cap):
    rng = np.random.default_rng(rows)
    A, W = rng.standard_normal((rows, 70)) * 4, bf16w(rng, 205, 70)
    got = gemm(ctx, dtype, CAP, A, W, out_f32=np.full((rows, 205), 7.0, np.float32), ld_out=205, cols=205, out_scale=scale, out_cap=cap)["out_f32"]
    close_to(got, pd.soft_cap(rounded(A, dtype) @ W.T.astype(np.float64) * scale, cap or None), "float32", factor=3)


# ---- experts -----------------------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("rows", [1, 40, 300])
@pytest.mark.parametrize("experts,top,job_rows", [(5, 2, 16), (130, 6, 32), (12, 12, 64), (1, 1, 128), (300, 1, 16)])
def test_choice_by_sigmoid_scores(ctx, rows, experts, top, job_rows):
    rng, bufs = np.random.default_rng(experts), []
    z = (rng.standard_normal((rows, experts)) * 2).astype(np.float32)
    z[0, :] = 0.25                                        # all equal: the lowest indices
    if rows > 1:
        z[1] = 20.0 + np.arange(experts) * 0.01           # sigmoids that are one in f32
    slots, jobs = (getattr(ctx.lib, n)(rows, experts, top, *r) for n, r in (("m40llm_ext_expert_slots", ()), ("m40llm_ext_expert_max_jobs", (job_rows,))))
    ids, weight, rows_of, place, job, slot_weight = (ctx.to_device(np.full(n, 77, t)) for n, t in ((rows * top, np.uint32), (rows * top, np.float32), (slots, np.uint32),
                                                                                                  (rows * top, np.uint32), (4 + 4 * jobs, np.uint32), (slots, np.float32)))
    call(ctx, "m40llm_ext_route_rows_async", C.byref(Route(rows=rows, experts=experts, top=top, job_rows=job_rows, score=1, scale=1.0, ld_logits=experts, logits=dev(ctx, bufs, z),
                                                           ids=ids.ptr, weight=weight.ptr, rows_of=rows_of.ptr, place=place.ptr, jobs=job.ptr, slot_weight=slot_weight.ptr)), 1)
    order = np.argsort(-z, axis=1, kind="stable")[:, :top]
    w = pd.sigmoid(np.take_along_axis(z, order, axis=1).astype(np.float64))
    assert np.array_equal(ids.download(np.uint32, (rows, top)), order)
    assert np.allclose(weight.download(np.float32, (rows, top)), w, rtol=3e-6)
    at, got, of = place.download(np.uint32, (rows, top)), slot_weight.download(np.float32, (slots,)), rows_of.download(np.uint32, (slots,))
    assert np.allclose(got[at], w, rtol=3e-6) and np.array_equal(of[at], np.repeat(np.arange(rows)[:, None], top, axis=1))
    used = job.download(np.uint32, (4 + 4 * jobs,))[1]
    assert np.all(np.delete(got[:used], np.unique(at)) == 0)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("job_rows,counts", [(16, [3, 0, 16, 20]), (32, [30, 33, 0, 1]), (64, [70, 5, 64, 0]), (128, [130, 0, 17, 140])])
def test_experts_take_weighted_inputs(ctx, dtype, job_rows, counts):
    if job_rows == 128 and dtype == "float32":
        pytest.skip("f32 jobs have up to 64 rows")
    rng, keep = np.random.default_rng(job_rows), []
    k, ff, limit, rows = 72, 40, 0.9, 150
    h = rng.standard_normal((rows, k)) * 1.5
    h[3] *= 20                                             # far beyond both limits
    W = [(bf16w(rng, ff, k), bf16w(rng, ff, k)) for _ in counts]
    tiles = []
    for a, b in W:                                         # gate and up tiles in turn
        ga, ub = (pack_tiles(ld.f32_to_bf16(np.concatenate([x, np.zeros((48 - ff, k), np.float32)]))).reshape(3, -1) for x in (a, b))
        tiles.append(np.stack([ga, ub], axis=1).reshape(-1))
    slots, jobs, rows_of, weight = 0, [], [], []
    for e, n in enumerate(counts):
        jobs += [(e, slots + j, min(job_rows, n - j), 0) for j in range(0, n, job_rows)]
        m = (n + 15) // 16 * 16
        rows_of += rng.integers(0, rows, size=m).tolist()
        weight += rng.uniform(0.1, 1.0, size=n).tolist() + [0.0] * (m - n)
        slots += m
    weight = np.array(weight, np.float32)
    plain = np.zeros((rows, up32(k)))
    plain[:, :k] = h
    d_rows = as_act(plain, dtype)
    table = np.concatenate([[len(jobs), slots, 0, 0], np.array(jobs).reshape(-1)])
    out = ctx.to_device(filled(slots * up32(ff), dtype))
    g = Gemm(act_dtype=ACT[dtype], epilogue=PROJECT, lda=up32(k), w=dev(ctx, keep, np.concatenate(tiles)), n_tiles=6, k_tiles=up32(k) // 32, w_batch=6 * up32(k) // 32 * 512, rows=rows,
             batches=1, out_act=out.ptr, ld_act=up32(ff), activation=LIMITED, act_alpha=1.702, act_limit=limit, row_scale=dev(ctx, keep, weight), jobs=u32(ctx, keep, table),
             max_jobs=len(jobs) + 2, job_rows=job_rows)
    if job_rows == 128:
        g.a = dev(ctx, keep, pack_tiles(d_rows[np.array(rows_of)]))
    else:
        g.a, g.gather = dev(ctx, keep, d_rows), u32(ctx, keep, rows_of)
    call(ctx, "m40llm_ext_packed_gemm_async", C.byref(g), 1)
    got = from_act(unpack_tiles(out.download(act_type(dtype), (slots * up32(ff),)), slots, up32(ff)), dtype)
    for e, first, n, _ in jobs:
        x = rounded(h, dtype)[np.array(rows_of[first:first + n])] * weight[first:first + n, None].astype(np.float64)
        close_to(got[first:first + n, :ff], pd.limited_gate(x @ W[e][0].T.astype(np.float64), x @ W[e][1].T.astype(np.float64), limit), dtype, factor=3)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows,width,top", [(5, 36, 1), (130, 256, 3), (17, 4100, 6)])
def test_one_stream_takes_experts_rows_as_they_are(ctx, dtype, rows, width, top):
    rng, keep = np.random.default_rng(width), []
    X, slots, ldo = rng.standard_normal((rows, width)).astype(np.float32), rows * top + 3, (width + 7) // 8 * 8
    out = np.zeros((slots, ldo))
    out[:, :width] = rng.standard_normal((slots, width))
    place = rng.permutation(slots)[:rows * top].reshape(rows, top)
    one, w, ldh = dev(ctx, keep, np.ones(1, np.float32)), (1 + 0.3 * rng.standard_normal(width)).astype(np.float32), up32(width)
    dx, h = ctx.to_device(X), ctx.to_device(filled((rows + 15) // 16 * 16 * ldh, dtype))
    call(ctx, "m40llm_ext_stream_update_async", C.byref(Update(act_dtype=ACT[dtype], rows=rows, width=width, streams=1, eps=0.1, mult=1.0, streams_x=dx.ptr, stream_stride=rows * width,
                                                               mix=one, share=one, take=one, expert_out=dev(ctx, keep, as_act(out, dtype)), ld_expert=ldo, top=top,
                                                               place=u32(ctx, keep, place), w=dev(ctx, keep, w), h=h.ptr, ld_h=ldh)), 1)
    x = X + rounded(out, dtype)[place][..., :width].sum(axis=1)
    close_to(dx.download(np.float32, X.shape), x, "float32", factor=2)
    close_to(from_act(unpack_tiles(h.download(act_type(dtype), ((rows + 15) // 16 * 16 * ldh,)), rows, ldh), dtype)[:, :width], pd.root_norm(x, 0.1) * w, dtype, factor=2)


# ---- attention -----------------------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,dim,vdim", [(4, 2, 64, 64), (3, 1, 21, 37), (9, 3, 10, 12), (1, 1, 1, 1), (2, 1, 256, 256), (16, 4, 128, 96)])
def test_heads_over_their_root_mean_square(ctx, dtype, H, G, dim, vdim):
    rng, keep = np.random.default_rng(dim + vdim), []
    eps, n = 0.2, 70
    slot, pos = [2] * n + [0] * n, 2 * list(range(n))
    rows = 2 * n
    k0 = (H * dim + 15) // 16 * 16
    v0 = k0 + (G * dim + 15) // 16 * 16
    cols = (v0 + G * vdim + 3) // 4 * 4
    proj = rng.standard_normal((rows, cols)).astype(np.float32) * np.repeat(np.exp(rng.standard_normal(rows)), cols).reshape(rows, cols).astype(np.float32)
    cache, pad = Cache(ctx, dtype, G, dim, vdim, 3, 2), up32(dim)
    dq = ctx.to_device(filled((rows, H, pad), dtype))
    call(ctx, "m40llm_ext_pair_split_append_async", C.byref(Split(
        act_dtype=ACT[dtype], rows=rows, maps=1, heads=H, kv_heads=G, dim=dim, vdim=vdim, eps=eps, proj=dev(ctx, keep, proj), ld_proj=cols, k_offset=k0, v_offset=v0,
        q_norm=dev(ctx, keep, np.full(dim, -1.0, np.float32)), k_norm=dev(ctx, keep, np.ones(dim, np.float32)), queries=dq.ptr, cache=cache.pages.ptr, row_slot=u32(ctx, keep, slot),
        row_pos=u32(ctx, keep, pos), row_back=u32(ctx, keep, [LONE] * rows), page_table=cache.d_table.ptr, max_pages=cache.max_pages)), 1)
    p = proj.astype(np.float64)
    got = from_act(dq.download(act_type(dtype), (rows, H, pad)), dtype)
    close_to(got[..., :dim], -pd.root_norm(p[:, :H * dim].reshape(rows, H, dim), eps), dtype)
    assert np.all(got[..., dim:] == 0)
    for i, sl in ((0, 2), (1, 0)):
        gk, gv = cache.read(sl, n)
        close_to(gk, pd.root_norm(p[i * n:(i + 1) * n, k0:k0 + G * dim].reshape(n, G, dim), eps), dtype)
        close_to(gv, p[i * n:(i + 1) * n, v0:v0 + G * vdim].reshape(n, G, vdim), dtype)


def attend(ctx, dtype, cache, cfg, q, slot, pos, portions, form, splits, tile_queries, scale, cap, window, slopes, sink, most=0.0, even=0):
    H, G, dim, vdim = cfg
    keep, rows, pad, group = [], len(q), up32(dim), H // G
    qq = np.zeros((rows, H, pad), np.float32)
    qq[..., :dim] = q
    size = 16 if form == 0 else tile_queries
    tiles = [(r * group + i, min(size, n * group - i)) for r, n in portions for i in range(0, n * group, size)]
    ctx.lib.m40llm_ext_pair_attention_partial_floats.restype = C.c_uint64
    floats = ctx.lib.m40llm_ext_pair_attention_partial_floats(1, rows, H, vdim, splits)
    partial, ldo = ctx.alloc(max(floats, 4) * 4), up32(H * vdim)
    out = ctx.to_device(filled((rows + 15) // 16 * 16 * ldo, dtype))
    a = Attn(act_dtype=ACT[dtype], form=form, maps=1, heads=H, kv_heads=G, dim=dim, vdim=vdim, scale=scale, out_scale=1.0, queries=dev(ctx, keep, as_act(qq, dtype)),
             cache=cache.pages.ptr, row_slot=u32(ctx, keep, slot), row_pos=u32(ctx, keep, pos), page_table=cache.d_table.ptr, max_pages=cache.max_pages, tiles=u32(ctx, keep, tiles),
             n_tiles=len(tiles), tile_queries=tile_queries, splits=splits, n_rows=rows, partial=partial.ptr, partial_floats=floats, out=out.ptr, ld_out=ldo, window=window or 0,
             cap=cap or 0.0, most=most, even=even, slopes=None if slopes is None else dev(ctx, keep, slopes, np.float32), sink=None if sink is None else dev(ctx, keep, sink, np.float32))
    call(ctx, "m40llm_ext_pair_attention_async", C.byref(a), 1)
    return from_act(unpack_tiles(out.download(act_type(dtype), ((rows + 15) // 16 * 16 * ldo,)), rows, ldo), dtype)[:, :H * vdim].reshape(rows, H, vdim)


def attend_want(q, k, v, pos, cfg, scale, cap, window, slopes, sink):
    H, G = cfg[:2]
    return np.stack([pd.attend_head(q[:, a], k[:, a // (H // G)], v[:, a // (H // G)], pos, scale, cap, 0.0 if slopes is None else np.float64(np.float32(slopes[a])), window,
                                    -1e30 if sink is None else np.float64(np.float32(sink[a]))) for a in range(H)], axis=1)


# cap, window, with slopes, sink's mean
OPTIONS = [(None, None, False, 2.0), (20.0, None, False, None), (None, 70, False, None), (None, None, True, None), (25.0, 64, True, 3.0), (30.0, 129, True, 25.0), (20.0, 1, True, 1.0),
           (22.0, 2, False, 0.0), (24.0, 100, True, -50.0)]


@pytest.mark.parametrize("dtype,form,splits,tile", FORMS)
@pytest.mark.parametrize("H,G,dim,vdim", [(4, 2, 64, 64), (3, 1, 20, 37), (8, 2, 128, 128), (1, 1, 1, 1), (2, 1, 160, 144), (17, 1, 33, 16)])
@pytest.mark.parametrize("cap,window,slopes,sink", OPTIONS)
def test_attention_with_keys_that_stand_out_at_the_edges(ctx, dtype, form, splits, tile, H, G, dim, vdim, cap, window, slopes, sink):
    """Every query row looks for one key: the oldest it sees, the one before that, itself, the one behind it, others at page borders.  Keys outside
    the window or the past would win if they were seen."""
    if form == 1 and ctx.lib.m40llm_ext_pair_attention_tile_queries(0, 1, dim, vdim) < tile:
        pytest.skip("these sizes have no such tile")
    rng = np.random.default_rng(dim + (window or 0))
    cfg, n, rows, scale = (H, G, dim, vdim), 330, 150, 0.8
    cache, kv = Cache(ctx, dtype, G, dim, vdim, 3, 6), {}
    for s in (0, 2):
        kv[s] = tuple(rounded(x, dtype) for x in (rng.standard_normal((n, G, dim)) * 0.3, rng.standard_normal((n, G, vdim))))
    cache.fill(ctx, kv)
    portions = [(0, 100), (100, 1), (101, rows - 101)]
    slot, pos = [2] * 100 + [0] + [2] * (rows - 101), list(range(200, 300)) + [n - 1] + list(range(20, 20 + rows - 101))
    w = window or n
    q = np.zeros((rows, H, dim))
    for r in range(rows):
        for a in range(H):
            p = pos[r]
            far = [max(p - w + 1, 0), max(p - w, 0), p, min(p + 1, n - 1), min(max(p - w + 2, 0), p), p // 64 * 64, max(p // 64 * 64 - 1, 0), int(rng.integers(0, p + 1)), 0][(r + a) % 9]
            key = kv[slot[r]][0][far, a // (H // G)]
            q[r, a] = key / (key @ key) * 30 if dim > 1 else key * 9
    q = rounded(q, dtype)
    m = 2.0 ** (-8.0 * (np.arange(H) + 1) / max(H, 2)) if slopes else None
    sinks = None if sink is None else sink + rng.standard_normal(H)
    args = (scale, cap, window, m, sinks)
    got = attend(ctx, dtype, cache, cfg, q, slot, pos, portions, form, splits, tile, *args)
    for first, c in portions:
        k, v = kv[slot[first]]
        close_to(got[first:first + c], attend_want(q[first:first + c], k, v, pos[first:first + c], cfg, *args), dtype, factor=4)


@pytest.mark.parametrize("dtype,form,splits,tile", FORMS)
@pytest.mark.parametrize("cap,window,slopes,sink", OPTIONS)
def test_attention_over_many_like_keys(ctx, dtype, form, splits, tile, cap, window, slopes, sink):
    """Flat scores: every key of the window counts, and the sink once."""
    rng = np.random.default_rng(3)
    cfg, n = (4, 2, 64, 128), 700
    cache = Cache(ctx, dtype, 2, 64, 128, 2, 11)
    k, v = rounded(rng.standard_normal((n, 2, 64)), dtype), rounded(rng.standard_normal((n, 2, 128)) + 0.5, dtype)
    cache.fill(ctx, {1: (k, v)})
    pos, q = np.arange(n - 70, n), rounded(rng.standard_normal((70, 4, 64)), dtype)
    args = (0.125, cap, window, 2.0 ** np.arange(-8, -4) if slopes else None, None if sink is None else sink + rng.standard_normal(4))
    got = attend(ctx, dtype, cache, cfg, q, [1] * 70, pos, [(0, 70)], form, splits, tile, *args)
    close_to(got, attend_want(q, k, v, pos, cfg, *args), dtype, factor=3)


@pytest.mark.parametrize("tile", [64, 128])
@pytest.mark.parametrize("even", [0, 1])
@pytest.mark.parametrize("H,G,dim,vdim", [(4, 2, 64, 64), (3, 1, 20, 37), (8, 2, 128, 128), (2, 1, 160, 144)])
@pytest.mark.parametrize("cap,window", [(3.0, None), (12.0, 65), (40.0, 200), (60.0, 100)])
def test_attention_of_bounded_products(ctx, H, G, dim, vdim, cap, window, tile, even):
    """Normed queries and keys, whose products are bounded: just inside the polynomial's range, where its error is largest, and beyond it."""
    if ctx.lib.m40llm_ext_pair_attention_tile_queries(0, 1, dim, vdim) < tile:
        pytest.skip("these sizes have no such tile")
    rng, n, rows = np.random.default_rng(dim), 330, 150
    cfg, cache = (H, G, dim, vdim), Cache(ctx, "bfloat16", G, dim, vdim, 1, 6)
    k, v = rounded(pd.root_norm(rng.standard_normal((n, G, dim)), 1e-6), "bfloat16"), rounded(rng.standard_normal((n, G, vdim)), "bfloat16")
    cache.fill(ctx, {0: (k, v)})
    pos = np.arange(n - rows, n)
    q = np.stack([k[np.maximum(pos - (7 * h) % 90, 0), h // (H // G)] * (-1) ** h for h in range(H)], axis=1)      # products of dim and minus dim
    m = 2.0 ** (-8.0 * (np.arange(H) + 1) / H)
    for reach in (0.49, 1.5):
        scale = reach * cap / (1.02 * dim)
        args = (scale, cap, window, m, rng.standard_normal(H))
        got = attend(ctx, "bfloat16", cache, cfg, q, [0] * rows, pos, [(0, rows)], 1, 1, tile, *args, most=1.02 * dim, even=even)
        close_to(got, attend_want(q, k, v, pos, cfg, *args), "bfloat16", factor=3)


def test_attention_refuses_what_only_one_map_has(ctx):
    b = ctx.alloc(1 << 16)
    ok = dict(maps=2, heads=1, kv_heads=1, dim=16, vdim=16, scale=1.0, ld_out=32, n_rows=1, n_tiles=1, splits=1,
              **{k: b.ptr for k in ("queries", "cache", "gate", "row_slot", "row_pos", "page_table", "tiles", "out")})
    for bad in (dict(window=3), dict(cap=1.0), dict(slopes=b.ptr), dict(sink=b.ptr), dict(maps=1, cap=-1.0), dict(maps=1, window=0x80000000), dict(maps=3)):
        call(ctx, "m40llm_ext_pair_attention_async", C.byref(Attn(**dict(ok, **bad))), 1, rc=-3)


# ---- row-wise steps --------------------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width,mixes", [(32, 5), (100, 1), (2100, 3)])
def test_rows_mixed_with_the_one_before(ctx, dtype, width, mixes):
    """Portions of one row and more over three slots, one of them fresh on an old state, again and again."""
    rng = np.random.default_rng(width)
    ldw = up32(width)
    mu = np.zeros((mixes, ldw), np.float32)
    mu[:, :width] = rng.uniform(-0.5, 1.5, (mixes, width))
    state = ctx.to_device(np.full((3, ldw), 5.0, np.float32))
    before, at = {0: np.zeros(ldw), 1: np.full(ldw, 5.0), 2: np.full(ldw, 5.0)}, {0: 0, 1: 9, 2: 77}
    for portions in ([(0, 1, 1), (1, 40, 0), (41, 2, 2)], [(0, 1, 2), (1, 1, 0)], [(0, 3, 2), (3, 130, 1), (133, 2, 0)]):
        keep, rows = [], sum(p[1] for p in portions)
        h = np.zeros((rows, ldw))
        h[:, :width] = rng.standard_normal((rows, width))
        hr = rounded(h, dtype)
        want, pos, back = np.zeros((rows, mixes, ldw)), [], []
        for r, n, s in portions:
            prev = pd.shifted(hr[r:r + n], before[s])
            for m in range(mixes):
                want[r:r + n, m] = pd.token_mix(hr[r:r + n], prev, mu[m].astype(np.float64))
            before[s] = hr[r + n - 1]
            pos += list(range(at[s], at[s] + n))
            back += [LONE] if n == 1 else list(range(n))
            at[s] += n
        out = ctx.to_device(filled((rows + 15) // 16 * 16 * mixes * ldw, dtype))
        call(ctx, "m40llm_ext_token_mix_async", C.byref(Mix(
            act_dtype=ACT[dtype], rows=rows, ld=ldw, mixes=mixes, h=dev(ctx, keep, as_act(h, dtype)), mu=dev(ctx, keep, mu), state=state.ptr, out=out.ptr,
            portions=u32(ctx, keep, [(r, n, s, 0) for r, n, s in portions]), row_pos=u32(ctx, keep, pos), row_back=u32(ctx, keep, back), n_portions=len(portions))), 1)
        got = from_act(unpack_tiles(out.download(act_type(dtype), ((rows + 15) // 16 * 16 * mixes * ldw,)), rows, mixes * ldw), dtype)
        close_to(got.reshape(rows, mixes, ldw), want, dtype)
        assert np.array_equal(state.download(np.float32, (3, ldw)), np.stack([before[s] for s in range(3)]))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows,cols", [(1, 1), (3, 40), (33, 320), (40, 13000), (1024, 100), (1030, 5632), (1025, 11500)])
def test_normed_polynomial(ctx, dtype, rows, cols):
    rng, ldz = np.random.default_rng(cols), up32(cols)
    act, eps = np.array([0.7, -1.2, 0.5, 0.3], np.float32), 0.05
    z = np.zeros((rows, ldz))
    z[:, :cols] = rng.standard_normal((rows, cols)) * np.exp(rng.standard_normal((rows, 1)))
    buf = ctx.to_device(pack_tiles(as_act(z, dtype)))
    call(ctx, "m40llm_ext_poly_norm_rows_async", buf.ptr, ldz, dev(ctx, keep := [], act), rows, cols, C.c_float(eps), ACT[dtype], 1)
    got = from_act(unpack_tiles(buf.download(act_type(dtype), ((rows + 15) // 16 * 16 * ldz,)), rows, ldz), dtype)
    assert np.all(got[:, cols:] == 0)
    want = pd.poly_norm(rounded(z[:, :cols], dtype), act.astype(np.float64), eps)
    assert np.abs(got[:, :cols] - want).max() < {"float32": 2e-5, "bfloat16": 5e-3}[dtype] * np.abs(want).max()
    for r in (0, rows - 1):
        close_to(got[r, :cols], want[r], dtype, factor=4)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows", [1, 40, 200])
@pytest.mark.parametrize("cols,groups", [(128, 2), (60, 4), (36, 36), (4096, 8), (4096, 1), (2200, 1), (4100, 2), (5000, 20), (1, 1)])
def test_gate_then_norm_over_parts(ctx, dtype, rows, cols, groups):
    rng, keep, eps = np.random.default_rng(cols), [], 0.1
    ldy, ldg, ldo = (cols + 3) // 4 * 4, (cols + 19) // 4 * 4, up32(cols)
    y, z, w = rng.standard_normal((rows, ldy)).astype(np.float32), rng.standard_normal((rows, ldg)).astype(np.float32) * 2, (1 + 0.3 * rng.standard_normal(cols)).astype(np.float32)
    y *= np.exp(rng.standard_normal((rows, ldy // 4)).repeat(4, axis=1)).astype(np.float32)
    out = ctx.to_device(filled((rows + 15) // 16 * 16 * ldo, dtype))
    call(ctx, "m40llm_ext_gate_group_norm_rows_async", dev(ctx, keep, y), C.c_uint64(ldy), dev(ctx, keep, z), C.c_uint64(ldg), dev(ctx, keep, w), rows, cols, groups, C.c_float(eps), out.ptr,
         ldo, ACT[dtype], 1)
    got = from_act(unpack_tiles(out.download(act_type(dtype), ((rows + 15) // 16 * 16 * ldo,)), rows, ldo), dtype)
    close_to(got[:, :cols], pd.gated_group_norm(y[:, :cols].astype(np.float64), z[:, :cols].astype(np.float64), groups, w, eps), dtype, factor=2)
    assert np.all(got[:, cols:] == 0)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,dim,vdim,taps", [(4, 2, 64, 128, 4), (6, 3, 20, 37, 3), (2, 2, 12, 8, 2), (1, 1, 1, 1, 1), (2, 1, 128, 96, 5), (2, 1, 256, 256, 3), (3, 1, 33, 20, 4)])
@pytest.mark.parametrize("cuts", [[70], [1] * 12, [2, 1, 3, 1, 1, 64, 2, 2, 130, 1]])
def test_convolution_with_bias_as_rows_of_heads(ctx, dtype, H, G, dim, vdim, taps, cuts):
    """Two sequences side by side, cut the same way, on a ring with old contents."""
    rng = np.random.default_rng(dim + taps)
    n, cols = sum(cuts), H * vdim + 2 * G * dim
    ldp, dp, vp = (cols + 3) // 4 * 4, up32(dim), up32(vdim)
    ldo = 2 * G * dp + H * vp
    u = rng.standard_normal((2, n, ldp)).astype(np.float32)
    W, b = rng.standard_normal((cols, taps)).astype(np.float32), rng.standard_normal(cols).astype(np.float32)
    state = ctx.to_device(np.full((3, max(taps - 1, 1), ldp), 99.0, np.float32))
    got, at = [[], []], 0
    for c in cuts:
        keep, proj, rows = [], np.concatenate([u[0, at:at + c], u[1, at:at + c]]), 2 * c
        slot, pos, back = [2] * c + [0] * c, 2 * list(range(at, at + c)), 2 * ([LONE] if c == 1 else list(range(c)))
        out = ctx.to_device(filled((rows + 15) // 16 * 16 * ldo, dtype))
        s = Space(act_dtype=ACT[dtype], rows=rows, heads=H, kv_heads=G, dim=dim, vdim=vdim, taps=taps, proj=dev(ctx, keep, proj), ld_proj=ldp, conv=dev(ctx, keep, W.T),
                  bias=dev(ctx, keep, b), conv_state=state.ptr, ld_state=ldp, out=out.ptr, ld_out=ldo, row_slot=u32(ctx, keep, slot), row_pos=u32(ctx, keep, pos), row_back=u32(ctx, keep, back))
        call(ctx, "m40llm_ext_space_split_async", C.byref(s), 1)
        if c > 1 and taps > 1:
            call(ctx, "m40llm_ext_conv_state_async", s.proj, C.c_uint64(ldp), cols, taps, state.ptr, C.c_uint64(ldp), u32(ctx, keep, [(0, c, 2, 0), (c, c, 0, 0)]), s.row_pos, 2, 1)
        y = from_act(unpack_tiles(out.download(act_type(dtype), ((rows + 15) // 16 * 16 * ldo,)), rows, ldo), dtype)
        for i in (0, 1):
            got[i].append(y[i * c:(i + 1) * c])
        at += c
    for i in (0, 1):
        y, _ = pd.short_convolution(u[i, :, :cols].astype(np.float64), np.zeros((taps - 1, cols)), W.astype(np.float64))
        x, B, Cq = np.split(pd.silu(y + b), [H * vdim, H * vdim + G * dim], axis=1)
        want = np.zeros((n, ldo))
        for part, first, k, size, pad in ((Cq, 0, G, dim, dp), (B, G * dp, G, dim, dp), (x, 2 * G * dp, H, vdim, vp)):
            want[:, first:first + k * pad].reshape(n, k, pad)[..., :size] = part.reshape(n, k, size)
        g = np.concatenate(got[i])
        close_to(g, want, dtype, factor=2)
        assert np.all(g[want == 0] == 0)


# ---- recurrences -----------------------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype,chunked", PATHS)
@pytest.mark.parametrize("H,dim", [(4, 64), (3, 20), (1, 1), (2, 128), (1, 256), (2, 130), (5, 33)])
@pytest.mark.parametrize("decays", ["long", "short", "mixed"])
def test_time_mixing(ctx, dtype, chunked, H, dim, decays):
    """Passes over three slots: a fresh portion on a slot with old contents, ones that go on, short ones that share their 64-row groups; channels that
    keep for hundreds of tokens, ones that lose all at once."""
    rng = np.random.default_rng(dim)
    eps, factor = 0.2, 0.6
    S = rng.standard_normal((3, H, dim, dim)).astype(np.float32).astype(np.float64)
    v4 = (dim + 3) // 4 * 4
    full = np.zeros((3, H, dim, v4), np.float32)
    full[..., :dim] = S
    state = ctx.to_device(full)
    w0 = {"long": rng.uniform(-7, -4, H * dim), "short": rng.uniform(0, 3, H * dim), "mixed": rng.choice([-9.0, -2.0, 6.0, 100.0], H * dim)}[decays].astype(np.float32)
    u, norm = rng.standard_normal(H * dim).astype(np.float32), (1 + 0.3 * rng.standard_normal(H * dim)).astype(np.float32)
    starts = {0: 0, 1: 7, 2: 500}
    for portions, what in RUNS:
        keep, rows, at, col = [], sum(p[1] for p in portions), 0, {}
        for c in "rkvg":
            col[c] = at + (3 if dim == 20 else 4)
            at = col[c] + (H * dim + 3) // 4 * 4
        rkv, z = rng.standard_normal((rows, at)).astype(np.float32), rng.standard_normal((rows, H * dim + 8)).astype(np.float32)
        p = {c: rkv[:, col[c]:col[c] + H * dim].astype(np.float64).reshape(rows, H, dim) for c in "rkvg"}
        with np.errstate(over="ignore"):
            w = pd.channel_decay(z[:, :H * dim].astype(np.float64) + w0).reshape(rows, H, dim)
        pos, want = np.zeros(rows, np.uint32), np.zeros((rows, H, dim))
        for r, n, s in portions:
            pos[r:r + n] = starts[s] + np.arange(n)
            cut = slice(r, r + n)
            want[cut], S[s] = pd.bonus_recurrence(p["r"][cut], p["k"][cut], p["v"][cut], w[cut], u.reshape(H, dim).astype(np.float64), S[s] if starts[s] else S[s] * 0)
            starts[s] += n
        want = factor * pd.root_norm(want, eps).reshape(rows, -1) * norm * pd.silu(p["g"].reshape(rows, -1))
        m = Mixing(heads=H, dim=dim, eps=eps, out_factor=factor, rkv=dev(ctx, keep, rkv), ld_rkv=at, decay=dev(ctx, keep, z), ld_decay=z.shape[1], w0=dev(ctx, keep, w0), u=dev(ctx, keep, u),
                   norm=dev(ctx, keep, norm), state=state.ptr, out_col=32, **{c + "_col": col[c] for c in "rkvg"})
        m.vdim = dim                                       # for the helper's scratch size; no field of the struct
        got = run_recurrence(ctx, keep, "m40llm_ext_time_mixing_async", m, 2, chunked, [(r, n, s, 0) for r, n, s in portions], pos, 32 + up32(H * dim), rows, dtype)
        close_to(got[:, 32:32 + H * dim], want, dtype, factor=20 if dtype == "float32" else 1)
        state_close(state.download(np.float32, full.shape)[..., :dim], S, chunked, what)


@pytest.mark.parametrize("dtype,chunked", PATHS)
@pytest.mark.parametrize("H,G,dim,vdim", [(4, 2, 64, 64), (6, 3, 20, 37), (1, 1, 1, 1), (8, 1, 128, 64), (2, 1, 256, 96), (2, 2, 256, 256), (3, 1, 33, 130), (4, 4, 48, 32)])
@pytest.mark.parametrize("decays", ["long", "short", "mixed"])
def test_stepped_linear_attention(ctx, dtype, chunked, H, G, dim, vdim, decays):
    rng = np.random.default_rng(dim + vdim)
    dp, vp = up32(dim), up32(vdim)
    S = rng.standard_normal((3, H, dim, vdim)).astype(np.float32).astype(np.float64)
    full = np.zeros((3, H, dim, vp), np.float32)
    full[..., :vdim] = S
    state = ctx.to_device(full)
    A_log = {"long": rng.uniform(-6, -3, H), "short": rng.uniform(0, 3, H), "mixed": rng.choice([-9.0, 0.0, 7.0], H)}[decays].astype(np.float32)
    bias, skip = rng.uniform(-2, 1, H).astype(np.float32), rng.standard_normal(H).astype(np.float32)
    starts, share = {0: 0, 1: 7, 2: 500}, np.arange(H) // (H // G)
    ctx.lib.m40llm_ext_lightning_scratch_bytes.restype = C.c_uint64
    for portions, what in RUNS:
        keep, rows = [], sum(p[1] for p in portions)
        ldq = 2 * G * dp + H * vp
        qkv = np.zeros((rows, ldq))
        q, k, v = (rounded(rng.standard_normal((rows, n, d)), dtype) for n, d in ((G, dim), (G, dim), (H, vdim)))
        for x, first, n, d, pad in ((q, 0, G, dim, dp), (k, G * dp, G, dim, dp), (v, 2 * G * dp, H, vdim, vp)):
            qkv[:, first:first + n * pad].reshape(rows, n, pad)[..., :d] = x
        z = (rng.standard_normal((rows, H + 3)) * 1.5).astype(np.float32)
        z[rows // 2] = 12.0
        dt = pd.softplus(z[:, :H].astype(np.float64) + bias)
        pos, want = np.zeros(rows, np.uint32), np.zeros((rows, H, vdim))
        for r, n, s in portions:
            pos[r:r + n] = starts[s] + np.arange(n)
            c = slice(r, r + n)
            want[c], S[s] = pd.space_recurrence(v[c], k[c][:, share], q[c][:, share], dt[c], pd.scalar_decay(dt[c], A_log.astype(np.float64)), skip.astype(np.float64),
                                                S[s] if starts[s] else S[s] * 0)
            starts[s] += n
        base, groups = [], []
        for i, (r, n, _) in enumerate(portions):
            base.append(len(groups))
            groups += [(i, g * 64) for g in range(r // 64, (r + n - 1) // 64 + 1)]
        nb = ctx.lib.m40llm_ext_lightning_scratch_bytes(len(groups), H, dim, vdim)
        scratch, ldo = ctx.to_device(np.full(nb // 4, np.nan, np.float32)), H * vdim + 2
        out = ctx.to_device(np.full((rows, ldo), 7.0, np.float32))
        call(ctx, "m40llm_ext_lightning_async", C.byref(Light(
            act_dtype=ACT[dtype], chunked=chunked, heads=H, dim=dim, vdim=vdim, kv_heads=G, qkv=dev(ctx, keep, pack_tiles(as_act(qkv, dtype))), ld_qkv=ldq, state=state.ptr, o=out.ptr,
            ld_o=ldo, portions=u32(ctx, keep, [(r, n, s, 0) for r, n, s in portions]), chunk_base=u32(ctx, keep, base), chunks=u32(ctx, keep, groups), row_pos=u32(ctx, keep, pos),
            n_portions=len(portions), n_chunks=len(groups), scratch=scratch.ptr, scratch_bytes=nb, step_logits=dev(ctx, keep, z), ld_step=H + 3, step_bias=dev(ctx, keep, bias),
            A_log=dev(ctx, keep, A_log), skip=dev(ctx, keep, skip))), 1)
        got = out.download(np.float32, (rows, ldo))
        assert np.all(got[:, H * vdim:] == 7.0)
        err = np.abs(got[:, :H * vdim].reshape(want.shape) - want).max() / np.abs(want).max()
        assert err < (6e-5 if chunked else 1e-5), (what, float(err))
        state_close(state.download(np.float32, full.shape)[..., :vdim], S, chunked, what)
