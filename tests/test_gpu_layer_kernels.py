"""The building blocks of layered decoders one by one, through the C ABI: packed products with each of their last steps, embedding,
norms, rotation, cache append, the two forms of latent attention, the greedy pick.  Inputs are made so that one key out of place, a
sink left out or counted twice, or a wrong page shows at once."""
import ctypes as C

import numpy as np
import pytest

pytestmark = pytest.mark.gpu

from pimosun_common import as_act, c_struct, close_to, from_act, ld, m40, pack_tiles, unpack_tiles, up32  # noqa: E402

Gemm, Split, Attn, Heads, Plan = (c_struct("M40llm" + n) for n in ("PackedGemm", "LatentSplit", "LatentAttention", "HeadAttention", "PackPlan"))
DTYPES = ["float32", "bfloat16"]
ACT = {"bfloat16": 0, "float32": 1}
STORE, ADD, STORE_ACT, GATED, ROTATE, PROJECT, KEYS, VALUES = range(8)
ROWS = [1, 2, 16, 17, 33, 64, 65, 129, 300]


@pytest.fixture(scope="module")
def ctx():
    yield m40.Context(0)


def call(ctx, name, *args, rc=0):
    got = getattr(ctx.lib, name)(ctx.h, *args)
    assert got == rc, (name, got)
    ctx.sync(1)


def act_type(dtype):
    return np.uint16 if dtype == "bfloat16" else np.float32


def rounded(a, dtype):
    return from_act(as_act(a, dtype), dtype).astype(np.float64)


def bf16w(rng, n, k, g=1.0):
    return ld.bf16_to_f32(ld.f32_to_bf16(rng.standard_normal((n, k)) * g / np.sqrt(k)))


def gemm(ctx, dtype, kind, A, W, out_f32=None, out_act=None, **kw):
    """A [rows][K] f32, W [N][K]; kw goes into the struct; buffers: numpy arrays that are uploaded and come back."""
    dA, dW = ctx.to_device(pack_tiles(as_act(A, dtype))), ctx.to_device(pack_tiles(ld.f32_to_bf16(W)))
    bufs = {"a": dA, "w": dW}
    g = Gemm(act_dtype=ACT[dtype], epilogue=kind, a=dA.ptr, lda=up32(A.shape[1]), w=dW.ptr, n_tiles=(W.shape[0] + 15) // 16,
             k_tiles=up32(W.shape[1]) // 32, rows=A.shape[0], batches=1)
    for k, v in dict(kw, out_f32=out_f32, out_act=out_act).items():
        if isinstance(v, np.ndarray):
            bufs[k] = ctx.to_device(v)
            v = bufs[k].ptr
        if v is not None:
            setattr(g, k, v)
    call(ctx, "m40llm_ext_packed_gemm_async", C.byref(g), 1)
    return {k: bufs[k].download(v.dtype, v.shape) for k, v in dict(out_f32=out_f32, out_act=out_act, rot_out=kw.get("rot_out")).items() if isinstance(v, np.ndarray)}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows", ROWS)
@pytest.mark.parametrize("n,k", [(50, 70), (128, 512), (257, 1100), (16, 32)])
def test_store_add_and_parts_of_k(ctx, dtype, rows, n, k):
    rng = np.random.default_rng(rows * 1000 + n)
    A, W = rng.standard_normal((rows, k)), bf16w(rng, n, k)
    want = rounded(A, dtype) @ W.T.astype(np.float64)
    for ld_out in (n, (n + 3) // 4 * 4 + 4):
        old = rng.standard_normal((rows, ld_out)).astype(np.float32)
        got = gemm(ctx, dtype, STORE, A, W, out_f32=old, ld_out=ld_out, cols=n)["out_f32"]
        close_to(got[:, :n], want, "float32", factor=2)
        assert np.array_equal(got[:, n:], old[:, n:])
        got = gemm(ctx, dtype, ADD, A, W, out_f32=old, ld_out=ld_out, cols=n)["out_f32"]
        close_to(got[:, :n], want + old[:, :n], "float32", factor=2)
        assert np.array_equal(got[:, n:], old[:, n:])
    tiles = up32(k) // 32
    for parts in (2, 3, 8):
        if (parts - 1) * ((tiles + parts - 1) // parts) >= tiles:
            continue
        got = gemm(ctx, dtype, STORE, A, W, out_f32=np.zeros((parts, rows, n), np.float32), ld_out=n, cols=n, k_parts=parts, out_batch=rows * n)["out_f32"]
        close_to(got.sum(axis=0), want, "float32", factor=2)
        assert np.abs(got).max(axis=(1, 2)).min() > 0


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows", [1, 20, 70, 200])
def test_products_per_head(ctx, dtype, rows):
    """STORE_ACT (plain rows) and GATED (packed, columns of a head that fill no group of four)."""
    rng = np.random.default_rng(rows)
    heads, k = 3, 64
    for n in (40, 37):
        A, W = rng.standard_normal((rows, heads * k)), [bf16w(rng, n, k) for _ in range(heads)]
        tiles = np.concatenate([pack_tiles(ld.f32_to_bf16(w)) for w in W])
        dA, dW = ctx.to_device(pack_tiles(as_act(A, dtype))), ctx.to_device(tiles)
        logits = rng.standard_normal((rows, 8)).astype(np.float32)
        gate = ctx.to_device(logits)
        want = np.stack([rounded(A[:, h * k:(h + 1) * k], dtype) @ W[h].T.astype(np.float64) for h in range(heads)], axis=1)
        for kind in (STORE_ACT, GATED):
            ldo = up32(heads * n)
            out = ctx.to_device(np.zeros((rows + 15) // 16 * 16 * ldo, act_type(dtype)))
            g = Gemm(act_dtype=ACT[dtype], epilogue=kind, a=dA.ptr, lda=heads * k, a_batch=k, w=dW.ptr, n_tiles=(n + 15) // 16, k_tiles=k // 32,
                     w_batch=(n + 15) // 16 * (k // 32) * 512, rows=rows, batches=heads, out_act=out.ptr, ld_act=ldo, act_batch=n, cols=n,
                     gate=gate.ptr, ld_gate=8)
            call(ctx, "m40llm_ext_packed_gemm_async", C.byref(g), 1)
            flat = out.download(act_type(dtype), ((rows + 15) // 16 * 16 * ldo,))
            got = from_act(flat.reshape(-1, ldo)[:rows] if kind == STORE_ACT else unpack_tiles(flat, rows, ldo), dtype)
            w = want if kind == STORE_ACT else want * (1 / (1 + np.exp(-logits[:, :heads, None].astype(np.float64))))
            close_to(got[:, :heads * n].reshape(rows, heads, n), w, dtype, factor=2)
            assert np.all(got[:, heads * n:] == 0)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows,split", [(5, 5), (40, 7), (100, 0), (200, 130)])
def test_rotated_queries(ctx, dtype, rows, split):
    rng = np.random.default_rng(rows)
    heads, dim, rot, k = 3, 40, 12, 96
    dp, rp = up32(dim), up32(rot)
    A = rng.standard_normal((rows, k))
    W = np.zeros((heads * (dp + rp), k), np.float32)
    w = bf16w(rng, heads * (dim + rot), k)
    for h in range(heads):
        W[h * (dp + rp):][:dim] = w[h * (dim + rot):][:dim]
        W[h * (dp + rp) + dp:][:rot] = w[h * (dim + rot) + dim:][:rot]
    spec = dict(dims=rot, base=300.0, scaling=dict(factor=3.0, original=40, fast=4.0, slow=0.5))
    pos = rng.integers(0, 5000, size=rows).astype(np.uint32)
    ang = angles(ctx, pos, spec, rp // 2)
    ldo = heads * (dp + rp)
    out = gemm(ctx, dtype, ROTATE, A, W, out_act=np.zeros((rows + 15) // 16 * 16 * ldo, act_type(dtype)), ld_act=ldo, head_width=dp + rp, rot_start=dp,
               heads=heads, split_row=split, rot_half=rp // 2, angles=ang, rot_out=np.zeros((rows, heads, rp + 32), act_type(dtype)), ld_rot=rp + 32)
    q = (rounded(A, dtype) @ w.T.astype(np.float64)).reshape(rows, heads, dim + rot)
    want = np.concatenate([q[:, :, :dim], ld.rotate(q[:, :, dim:], pos, spec)], axis=2)
    got = from_act(unpack_tiles(out["out_act"], rows, ldo), dtype).reshape(rows, heads, dp + rp)
    turned = from_act(out["rot_out"], dtype)
    close_to(got[:, :, :dim], want[:, :, :dim], dtype, factor=2)
    close_to(np.concatenate([turned[:split, :, :rot], got[split:, :, dp:dp + rot]]), want[:, :, dim:], dtype, factor=2)
    assert np.all(turned[:split, :, rot:] == 0) and np.all(turned[split:] == 0)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows", [1, 30, 64, 150, 500])
@pytest.mark.parametrize("ff,plain", [(23, 50), (160, 0), (600, 32)])
def test_projection_with_gated_feed_forward(ctx, dtype, rows, ff, plain):
    rng = np.random.default_rng(rows + ff)
    k = 100
    A, wp, wg, wu = rng.standard_normal((rows, k)), bf16w(rng, max(plain, 1), k), bf16w(rng, ff, k, 3.0), bf16w(rng, ff, k)
    P, F = (plain + 31) // 32 * 32, (ff + 15) // 16 * 16
    W = np.zeros((P + 2 * F, k), np.float32)
    W[:plain] = wp[:plain]
    for i in range(ff):
        W[P + i // 16 * 32 + i % 16] = wg[i]
        W[P + i // 16 * 32 + 16 + i % 16] = wu[i]
    col, ldo = 36, up32(36 + F)
    out = gemm(ctx, dtype, PROJECT, A, W, out_f32=np.zeros((rows, max(P, 4)), np.float32), ld_out=max(P, 4), out_act=np.zeros((rows + 15) // 16 * 16 * ldo, act_type(dtype)),
               ld_act=ldo, act_col=col, plain_tiles=P // 16)
    a = rounded(A, dtype)
    if plain:
        close_to(out["out_f32"][:, :plain], a @ wp.T.astype(np.float64), "float32", factor=2)
    got = from_act(unpack_tiles(out["out_act"], rows, ldo), dtype)
    close_to(got[:, col:col + ff], ld.gelu_tanh(a @ wg.T.astype(np.float64)) * (a @ wu.T.astype(np.float64)), dtype, factor=2)
    assert np.all(got[:, :col] == 0) and np.all(got[:, col + ff:] == 0)


def test_products_refuse_what_they_do_not_serve(ctx):
    b = ctx.alloc(1 << 16)
    ok = dict(act_dtype=0, epilogue=STORE, a=b.ptr, lda=64, w=b.ptr, n_tiles=2, k_tiles=2, rows=4, batches=1, out_f32=b.ptr, ld_out=32, cols=32)
    for bad, rc in ((dict(rows=0), -3), (dict(lda=40), -3), (dict(lda=32), -3), (dict(act_dtype=2), -3), (dict(epilogue=12), -3), (dict(segment_tiles=8), -3), (dict(segment_tiles=16, n_tiles=17, a_batch=64), -3),
                    (dict(segment_tiles=16, batches=2), -3), (dict(epilogue=11, out_cap=-1.0), -4), (dict(cols=33), -4),
                    (dict(k_parts=3), -3), (dict(k_parts=2, epilogue=ADD), -3), (dict(out_f32=None), -4), (dict(a=None), -1),
                    (dict(epilogue=KEYS, out_act=b.ptr, rows=64), -4), (dict(epilogue=GATED, out_act=b.ptr, ld_act=30), -3)):
        call(ctx, "m40llm_ext_packed_gemm_async", C.byref(Gemm(**dict(ok, **bad))), 1, rc=rc)
    h = Heads(heads=1, plain_tiles=1, rot_tiles=1, entry_tiles=2, vdim=16, v_tiles=1, ld_queries=64, n_jobs=1, job_rows=100, ld_out=32,
              **{n: b.ptr for n in ("queries", "keys", "values", "cache", "sink", "gate", "row_pos", "pages", "jobs", "out")})
    call(ctx, "m40llm_ext_head_attention_async", C.byref(h), 1, rc=-3)
    a = Attn(heads=1, kv_rank=32, latent_pad=32, entry_width=64, n_tiles=1, m_tiles=8, splits=1, n_queries=1,
             **{n: b.ptr for n in ("queries", "cache", "sink", "row_slot", "row_pos", "page_table", "tiles", "out")})
    call(ctx, "m40llm_ext_latent_attention_async", C.byref(a), 1, rc=-3)
    a.m_tiles, a.splits = 1, 2
    call(ctx, "m40llm_ext_latent_attention_async", C.byref(a), 1, rc=-4)


@pytest.mark.parametrize("width", [8, 80, 100, 4096])
def test_embedding_with_token_pairs(ctx, width):
    rng = np.random.default_rng(width)
    vocab, buckets, mp, mc = 50, 13, 4000000007, 3999999979
    E, B = rng.standard_normal((vocab, width)), rng.standard_normal((buckets + 1, width))
    toks = rng.integers(0, vocab, size=30).astype(np.uint32)
    prev = rng.integers(0, vocab, size=30).astype(np.uint32)
    prev[[0, 7]] = 0xffffffff
    dE, dB, dt, dp = (ctx.to_device(x) for x in (ld.f32_to_bf16(E), ld.f32_to_bf16(B), toks, prev))
    out = ctx.alloc(30 * width * 4)
    e, b = ld.bf16_to_f32(ld.f32_to_bf16(E)), ld.bf16_to_f32(ld.f32_to_bf16(B))
    for pairs in (True, False):
        call(ctx, "m40llm_ext_embed_pairs_async", dE.ptr, dB.ptr if pairs else None, dt.ptr, dp.ptr, 30, vocab, width, buckets, mp, mc, out.ptr, 1)
        rows = [ld.bigram_row(None if p == 0xffffffff else int(p), int(t), buckets, mp, mc) for p, t in zip(prev, toks)]
        want = e[toks] + (b[rows] if pairs else 0)
        assert np.array_equal(out.download(np.float32, (30, width)), want.astype(np.float32))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width", [1, 80, 100, 2048, 4100, 5000])
def test_layer_norm_rows_and_planes(ctx, dtype, width):
    rng = np.random.default_rng(width)
    rows, eps = 150, 2e-2
    x = (rng.standard_normal((rows, width)) * 0.2 + 3.0).astype(np.float32)      # a mean far from zero, a spread near eps
    planes = rng.standard_normal((3, rows, width)).astype(np.float32) * 0.1
    w = rng.standard_normal(width).astype(np.float32)
    index = rng.integers(0, rows, size=20).astype(np.uint32)
    ldo = up32(width)
    dP, dw, di = ctx.to_device(planes), ctx.to_device(w), ctx.to_device(index)
    for n_planes, use_index in ((0, False), (3, False), (3, True), (1, False)):
        dx = ctx.to_device(x)
        n = 20 if use_index else rows
        out = ctx.alloc((n + 15) // 16 * 16 * ldo * 4)
        call(ctx, "m40llm_ext_layer_norm_rows_async", dx.ptr, dP.ptr, n_planes, rows * width, dw.ptr, di.ptr if use_index else None, n, width, eps,
             out.ptr, ldo, ACT[dtype], 1)
        full = x.astype(np.float64) + planes[:n_planes].sum(axis=0, dtype=np.float64)
        got = from_act(unpack_tiles(out.download(act_type(dtype), ((n + 15) // 16 * 16 * ldo,)), n, ldo), dtype)
        close_to(got[:, :width], ld.layer_norm(full[index] if use_index else full, w, eps), dtype, factor=5 if dtype == "float32" else 1)
        assert np.all(got[:, width:] == 0)
        after = dx.download(np.float32, (rows, width))
        assert np.array_equal(after, x) if use_index or not n_planes else np.allclose(after, full, rtol=1e-6, atol=1e-6)


def angles(ctx, pos, spec, half):
    f, mag = ld.rotation(spec)
    dpos, df = ctx.to_device(np.asarray(pos, np.uint32)), ctx.to_device(f)
    out = ctx.alloc(len(pos) * half * 8)
    call(ctx, "m40llm_ext_rotation_angles_async", dpos.ptr, len(pos), df.ptr, len(f), half, mag, out.ptr, 1)
    return out.download(np.float32, (len(pos), half, 2))


@pytest.mark.parametrize("spec", [dict(dims=2, base=7.0), dict(dims=64, base=1e6, scaling=dict(factor=40.0, original=4096, fast=32.0, slow=1.0)),
                                  dict(dims=30, base=1e4, scaling=dict(factor=1.0, original=8, fast=1.0, slow=1.0))])
def test_rotation_angles_far_out(ctx, spec):
    pos = np.array([0, 1, 63, 64, 4095, 131071, 4000000000], np.uint32)
    half = up32(spec["dims"]) // 2
    got = angles(ctx, pos, spec, half)
    f, mag = ld.rotation(spec)
    a = pos.astype(np.float64)[:, None] * f
    assert np.abs(got[:, :len(f), 0] - np.cos(a) * mag).max() < 1e-6 * mag and np.abs(got[:, :len(f), 1] - np.sin(a) * mag).max() < 1e-6 * mag
    assert np.all(got[:, len(f):] == [1.0, 0.0])


def page_layout(entries, table, n_pages, width):
    """[tokens][width] entries of one sequence -> pages as they lie in memory (pages elsewhere: large finite values)."""
    pages = np.full((n_pages, 64 * width), 3.0, dtype=np.float64)
    for p, page in enumerate(table):
        e = np.full((64, width), -2.0)
        part = entries[p * 64:(p + 1) * 64]
        e[:len(part)] = part
        pages[page] = pack_tiles(e)
    return pages


@pytest.mark.parametrize("dtype", DTYPES)
def test_split_norm_rotate_append(ctx, dtype):
    rng = np.random.default_rng(1)
    rows, qr, kr, rd = 140, 37, 45, 10
    kv_off, rot_off = 48, 96
    ldp, lat, half = 128, up32(kr), 16
    ew = lat + 32
    proj = rng.standard_normal((rows, ldp)).astype(np.float32) * 0.1
    qn, kn = rng.standard_normal(qr).astype(np.float32), rng.standard_normal(kr).astype(np.float32)
    spec, eps = dict(dims=rd, base=50.0), 5e-3
    slot = np.repeat([2, 0], [100, 40]).astype(np.uint32)
    pos = np.concatenate([np.arange(30, 130), np.arange(60, 100)]).astype(np.uint32)
    table = np.zeros((3, 4), np.uint32)
    table[2, :3], table[0, :2] = [5, 1, 3], [0, 7]
    cache = np.full((8, 64 * ew), 9.0)
    bufs = {k: ctx.to_device(v) for k, v in dict(proj=proj, q_norm=qn, kv_norm=kn, cache=as_act(cache, dtype), cq=np.zeros(144 * up32(qr), act_type(dtype)),
                                                 angles=angles(ctx, pos, spec, half), row_slot=slot, row_pos=pos, page_table=table).items()}
    s = Split(act_dtype=ACT[dtype], rows=rows, ld_proj=ldp, q_rank=qr, kv_offset=kv_off, kv_rank=kr, rot_offset=rot_off, rot_dim=rd, eps=eps, ld_cq=up32(qr),
              latent_pad=lat, entry_width=ew, rot_half=half, max_pages=4, **{k: b.ptr for k, b in bufs.items()})
    call(ctx, "m40llm_ext_latent_split_append_async", C.byref(s), 1)
    p64 = proj.astype(np.float64)
    got = from_act(unpack_tiles(bufs["cq"].download(act_type(dtype), (144 * up32(qr),)), rows, up32(qr)), dtype)
    close_to(got[:, :qr], ld.rms_norm(p64[:, :qr], qn, eps), dtype)
    assert np.all(got[:, qr:] == 0)
    pages = from_act(bufs["cache"].download(act_type(dtype), cache.shape), dtype)
    want = np.full((8, 64, ew), 9.0)
    lat_want = ld.rms_norm(p64[:, kv_off:kv_off + kr], kn, eps)
    rot_want = ld.rotate(p64[:, rot_off:rot_off + rd], pos, spec)
    for i in range(rows):
        e = want[table[slot[i], pos[i] // 64], pos[i] % 64]
        e[:] = 0
        e[:kr], e[lat:lat + rd] = lat_want[i], rot_want[i]
    for p in range(8):
        close_to(unpack_tiles(pages[p], 64, ew), want[p], dtype, scale=np.abs(lat_want).max(), factor=1 if dtype == "bfloat16" else 2)


# ---- attention -------------------------------------------------------------------------------------------------------------


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,rank,rot", [(3, 40, 8), (16, 128, 32), (40, 64, 64), (5, 512, 64), (20, 512, 64), (33, 512, 64), (2, 700, 20)])
@pytest.mark.parametrize("splits", [1, 3, 16])
def test_latent_attention_finds_the_key_it_asks_for(ctx, dtype, heads, rank, rot, splits):
    """Two sequences on scattered pages: a portion of single tokens and a portion of several.  Query (row, head) asks for one position:
    first, last visible, page borders, far back -- or for one just out of sight, which must not be seen."""
    rng = np.random.default_rng(heads + rank)
    lat, rp = up32(rank), up32(rot)
    ew = lat + rp
    lens, firsts = [391, 200], [390, 197]
    tables = [[7, 2, 9, 0, 5, 11, 4], [3, 8, 1, 10]]
    rows_pos = np.array([390, 197, 198, 199], np.uint32)
    slot = np.array([1, 0, 0, 0], np.uint32)
    max_pages = 7
    table = np.zeros((2, max_pages), np.uint32)
    table[1, :7], table[0, :4] = tables[0], tables[1]
    entries, queries = [], []
    for n in lens:
        E = np.zeros((n, ew))
        E[:, :rank], E[:, lat:lat + rot] = rng.standard_normal((n, rank)) * 0.5, rng.standard_normal((n, rot)) * 0.5
        entries.append(rounded(E, dtype))
    cache = page_layout(entries[0], tables[0], 12, ew)
    second = page_layout(entries[1], tables[1], 12, ew)
    cache[tables[1]] = second[tables[1]]
    scale = 0.7
    sink = rng.standard_normal(heads).astype(np.float32)
    Q = np.zeros((4, heads, ew))
    for i in range(4):
        E, last = entries[0 if slot[i] == 1 else 1], int(rows_pos[i])
        spots = [0, last, 63, 64, 127, 128, last - 1, 1, 65, min(last + 1, len(E) - 1), 191, 192 if last >= 192 else 5]
        for h in range(heads):
            e = E[spots[h % len(spots)]]
            Q[i, h] = e * ((14.0 if h % 3 else 4.0) / scale / (e @ e))
    Q = rounded(Q, dtype)
    want = np.zeros((4, heads, rank))
    for i in range(4):
        E = entries[0 if slot[i] == 1 else 1][:int(rows_pos[i]) + 1]
        for h in range(heads):
            want[i, h] = ld.sink_softmax_attend((E @ Q[i, h]) * scale, E[:, :rank], sink[h])
    bufs = {k: ctx.to_device(v) for k, v in dict(queries=as_act(Q, dtype), cache=as_act(cache, dtype), sink=sink, row_slot=slot, row_pos=rows_pos,
                                                 page_table=table, out=np.zeros(16 * heads * lat, act_type(dtype))).items()}
    most = ctx.lib.m40llm_ext_latent_attention_max_m_tiles(ACT[dtype], rank, ew)
    assert most >= 1
    for mt in (1, 2, 4):
        if mt > most:
            continue
        tiles = []
        for row, n in ((0, 1), (1, 3)):
            for i in range(0, n * heads, 16 * mt):
                tiles += [row * heads + i, min(16 * mt, n * heads - i)]
        dt = ctx.to_device(np.array(tiles, np.uint32))
        need = ctx.lib.m40llm_ext_latent_attention_partial_floats(4 * heads, lat, splits)
        part = ctx.alloc(max(need, 1) * 4)
        a = Attn(act_dtype=ACT[dtype], heads=heads, kv_rank=rank, latent_pad=lat, entry_width=ew, scale=scale, max_pages=max_pages, tiles=dt.ptr,
                 n_tiles=len(tiles) // 2, m_tiles=mt, splits=splits, first_query=0, n_queries=4 * heads, partial=part.ptr, partial_floats=need,
                 **{k: b.ptr for k, b in bufs.items()})
        call(ctx, "m40llm_ext_latent_attention_async", C.byref(a), 1)
        got = from_act(unpack_tiles(bufs["out"].download(act_type(dtype), (16 * heads * lat,)), 4, heads * lat), dtype).reshape(4, heads, lat)
        close_to(got[:, :, :rank], want, dtype, factor=2)


@pytest.mark.parametrize("heads,dim,rot,vdim,rank,job_rows", [(3, 24, 8, 20, 40, 64), (2, 128, 64, 128, 512, 128), (5, 32, 32, 33, 64, 128),
                                                              (2, 150, 40, 100, 96, 64), (4, 1, 2, 1, 1, 64), (3, 100, 60, 64, 160, 64),
                                                              (2, 64, 32, 72, 64, 128), (1, 180, 40, 128, 128, 128)])
def test_head_attention_with_keys_and_values_from_pages(ctx, heads, dim, rot, vdim, rank, job_rows):
    """KEYS, VALUES and the attention over them: two sequences on scattered pages, a whole prompt and a portion behind a long context.
    Queries ask for positions at page borders, far back, the first, the last visible, and the next one, which must stay unseen."""
    rng = np.random.default_rng(heads * 7 + dim)
    dp, rp, lat, vt = up32(dim), up32(rot), up32(rank), (vdim + 15) // 16
    ew, qw = lat + rp, dp + rp
    specs = [([6, 0, 9, 3], 0, 210), ([5, 1, 8, 2, 7], 133, 170)]          # pages, tokens before, tokens of the portion
    cache, list_, entries, rows_pos, jobs, first_page = np.full((10, 64 * ew), 1.5), [], [], [], [], []
    for pages, before, n in specs:
        E = np.zeros((before + n, ew))
        E[:, :rank], E[:, lat:lat + rot] = rng.standard_normal((before + n, rank)), rng.standard_normal((before + n, rot)) * 0.5
        E = rounded(E, "bfloat16")
        entries.append(E)
        cache[pages] = page_layout(E, pages, 10, ew)[pages]
        for i in range(0, n, job_rows):
            jobs.append([len(rows_pos) + i, min(job_rows, n - i), len(list_), 0])
        list_ += pages
        rows_pos += list(range(before, before + n))
    Wk, Wv = bf16w(rng, heads * dim, rank), bf16w(rng, heads * vdim, rank)
    wk = np.zeros((heads * dp, rank), np.float32)
    wv = np.zeros((heads * vt * 16, rank), np.float32)
    for h in range(heads):
        wk[h * dp:][:dim], wv[h * vt * 16:][:vdim] = Wk[h * dim:][:dim], Wv[h * vdim:][:vdim]
    dc, dl = ctx.to_device(as_act(cache, "bfloat16")), ctx.to_device(np.array(list_, np.uint32))
    T = 64 * len(list_)
    keys, values = ctx.alloc(T * heads * dp * 2), ctx.alloc(T * heads * vt * 16 * 2)
    for kind, W, out in ((KEYS, wk, keys), (VALUES, wv, values)):
        dW = ctx.to_device(pack_tiles(ld.f32_to_bf16(W)))
        g = Gemm(act_dtype=0, epilogue=kind, a=dc.ptr, w=dW.ptr, n_tiles=W.shape[0] // 16, k_tiles=lat // 32, rows=T, batches=1, out_act=out.ptr,
                 pages=dl.ptr, page_k_tiles=ew // 32)
        call(ctx, "m40llm_ext_packed_gemm_async", C.byref(g), 1)
    scale = 0.6
    sink = (rng.standard_normal(heads) * 3).astype(np.float32)
    R = len(rows_pos)
    logits = rng.standard_normal((R, heads)).astype(np.float32)
    Q, want, at = np.zeros((R, heads, qw)), np.zeros((R, heads, vdim)), 0
    for (pages, before, n), E in zip(specs, entries):
        K = rounded((E[:, :rank] @ Wk.T.astype(np.float64)), "bfloat16").reshape(-1, heads, dim)
        V = rounded((E[:, :rank] @ Wv.T.astype(np.float64)), "bfloat16").reshape(-1, heads, vdim)
        for i in range(n):
            last = before + i
            spots = [s for s in (0, last, 63, 64, 127, 128, last - 1, last - 64, 191, 1) if 0 <= s <= last] + [min(last + 1, before + n - 1)]
            for h in range(heads):
                t = spots[(i + h) % len(spots)]
                k = np.concatenate([K[t, h], E[t, lat:lat + rot]])
                q = k * ((12.0 if i % 2 else 3.0) / scale / (k @ k))
                q = rounded(q, "bfloat16")
                Q[at + i, h, :dim], Q[at + i, h, dp:dp + rot] = q[:dim], q[dim:]
                s = (K[:last + 1, h] @ q[:dim] + E[:last + 1, lat:lat + rot] @ q[dim:]) * scale
                want[at + i, h] = ld.sink_softmax_attend(s, V[:last + 1, h], sink[h]) * ld.sigmoid(float(logits[at + i, h]))
        at += n
    ldo = up32(heads * vdim)
    bufs = {k: ctx.to_device(v) for k, v in dict(queries=pack_tiles(as_act(Q.reshape(R, -1), "bfloat16")), sink=sink, gate=logits, row_pos=np.array(rows_pos, np.uint32),
                                                 jobs=np.array(jobs, np.uint32), out=np.zeros((R + 15) // 16 * 16 * ldo, np.uint16)).items()}
    a = Heads(heads=heads, plain_tiles=dp // 32, rot_tiles=rp // 32, entry_tiles=ew // 32, vdim=vdim, v_tiles=vt, scale=scale, ld_queries=heads * qw,
              keys=keys.ptr, values=values.ptr, cache=dc.ptr, ld_gate=heads, pages=dl.ptr, n_jobs=len(jobs), job_rows=job_rows, ld_out=ldo,
              **{k: b.ptr for k, b in bufs.items()})
    call(ctx, "m40llm_ext_head_attention_async", C.byref(a), 1)
    got = from_act(unpack_tiles(bufs["out"].download(np.uint16, ((R + 15) // 16 * 16 * ldo,)), R, ldo), "bfloat16")
    close_to(got[:, :heads * vdim].reshape(R, heads, vdim), want, "bfloat16", factor=2)
    assert np.all(got[:, heads * vdim:] == 0)


def test_sink_counts_once_and_only_in_the_denominator(ctx):
    """One key of weight e^0 against sinks far below, equal and far above: results 1, 1/2, 0 times the latent, however the pages are split."""
    rank, ew, heads = 32, 64, 3
    E = np.zeros((100, ew))
    E[0, :rank] = 2.0
    sink = np.array([-80.0, 0.0, 80.0], np.float32)
    cache = page_layout(E, [1, 0], 2, ew)
    for dtype in DTYPES:
        bufs = {k: ctx.to_device(v) for k, v in dict(queries=as_act(np.zeros((1, heads, ew)), dtype), cache=as_act(cache, dtype), sink=sink,
                                                     row_slot=np.zeros(1, np.uint32), row_pos=np.zeros(1, np.uint32),
                                                     page_table=np.array([[1, 0]], np.uint32), tiles=np.array([0, heads], np.uint32),
                                                     out=np.zeros(16 * heads * rank, act_type(dtype))).items()}
        for splits in (1, 2):
            need = ctx.lib.m40llm_ext_latent_attention_partial_floats(heads, rank, splits)
            part = ctx.alloc(max(need, 1) * 4)
            a = Attn(act_dtype=ACT[dtype], heads=heads, kv_rank=rank, latent_pad=rank, entry_width=ew, scale=1.0, max_pages=2, n_tiles=1, m_tiles=1, splits=splits,
                     n_queries=heads, partial=part.ptr, partial_floats=need, **{k: b.ptr for k, b in bufs.items()})
            call(ctx, "m40llm_ext_latent_attention_async", C.byref(a), 1)
            got = from_act(unpack_tiles(bufs["out"].download(act_type(dtype), (16 * heads * rank,)), 1, heads * rank), dtype).reshape(heads, rank)
            assert np.allclose(got, np.array([2.0, 1.0, 0.0])[:, None], atol=1e-6), (dtype, splits, got[:, 0])


@pytest.mark.parametrize("vocab", [1, 31, 33, 5000])
def test_greedy_pick_ties_and_gap(ctx, vocab):
    rng = np.random.default_rng(vocab)
    rows, cap = 5, 3
    L = rng.standard_normal((rows, vocab)).astype(np.float32)
    if vocab > 31:
        L[1, [30, 7, vocab - 1]] = 50.0                  # a tie in different parts: the lowest index, gap 0
        L[2, :] = -np.inf
        L[2, 29] = -3.0
    dl, parts = ctx.to_device(L), ctx.alloc(rows * 32 * 16)
    tok = np.arange(rows).astype(np.uint32)
    b = [ctx.to_device(x) for x in (tok, np.full(rows, 0xffffffff, np.uint32), np.full(rows, 9, np.uint32), np.zeros(4, np.uint32),
                                    np.zeros((rows, cap), np.uint32), np.zeros((rows, cap), np.float32))]
    for step in range(2):
        call(ctx, "m40llm_ext_top2_parts_async", dl.ptr, rows, vocab, parts.ptr, 1)
        call(ctx, "m40llm_ext_advance_rows_async", parts.ptr, rows, *[x.ptr for x in b], cap, 1)
    ids, gaps = b[4].download(np.uint32, (rows, cap)), b[5].download(np.float32, (rows, cap))
    assert np.array_equal(ids[:, 0], L.argmax(axis=1)) and np.array_equal(ids[:, 1], ids[:, 0])
    if vocab > 1:
        srt = np.sort(L, axis=1)
        assert np.array_equal(gaps[:, 0], srt[:, -1] - srt[:, -2])
    assert np.array_equal(b[0].download(np.uint32, (rows,)), ids[:, 0]) and np.array_equal(b[1].download(np.uint32, (rows,)), ids[:, 0])
    assert np.all(b[2].download(np.uint32, (rows,)) == 11) and b[3].download(np.uint32, (4,))[0] == 2
