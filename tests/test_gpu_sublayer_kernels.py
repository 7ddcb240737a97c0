"""The building blocks of layers with norms on their outputs one by one, through the C ABI: embedding with positions, norm and add, norm and
gate, routing and products per expert, convolution with query and key norms, differential attention in its forms, lightning attention in
its forms.  Inputs are made so that one key out of place, a lost state, a wrong expert or a decay off by one token shows at once."""
import ctypes as C

import numpy as np
import pytest

pytestmark = pytest.mark.gpu

from gulidra_common import od  # noqa: E402
from pimosun_common import as_act, c_struct, close_to, from_act, ld, m40, pack_tiles, unpack_tiles, up32  # noqa: E402
from test_gpu_layer_kernels import ACT, DTYPES, PROJECT, STORE_ACT, act_type, bf16w, call, gemm, rounded  # noqa: E402

Embed, NormAdd, Route, Split, Attn, Light, Gemm = (c_struct("M40llm" + n) for n in ("EmbedTokens", "NormAdd", "Route", "PairSplit", "PairAttention",
                                                                                   "Lightning", "PackedGemm"))
SILU_KIND, SILU, INPUT, RMS = 8, 1, 0xffffffff, 1
LONE = 0x80000000


@pytest.fixture(scope="module")
def ctx():
    yield m40.Context(0)


def dev(ctx, keep, a, dtype=None):
    keep.append(ctx.to_device(np.ascontiguousarray(a, dtype=dtype)))
    return keep[-1].ptr


def u32(ctx, keep, a):
    return dev(ctx, keep, a, np.uint32)


def filled(shape, dtype):
    """An output buffer whose untouched elements show."""
    return np.full(shape, 0x4b4b if dtype == "bfloat16" else 12345.0, act_type(dtype))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows,width", [(1, 8), (5, 36), (130, 257), (300, 1024)])
def test_embedding_with_scale_and_positions(ctx, rows, width, dtype):
    rng, keep = np.random.default_rng(rows), []
    E, P = (ld.f32_to_bf16(rng.standard_normal((n, width))) for n in (40, 50))
    tok, pos = rng.integers(0, 40, rows), rng.integers(0, 50, rows)
    ldh = up32(width)
    x, h = ctx.to_device(np.zeros((rows, width), np.float32)), ctx.to_device(filled((rows + 15) // 16 * 16 * ldh, dtype))
    e = Embed(act_dtype=ACT[dtype], rows=rows, vocab=40, width=width, table=dev(ctx, keep, E), pos_table=dev(ctx, keep, P), tokens=u32(ctx, keep, tok),
              positions=u32(ctx, keep, pos), n_positions=50, scale=3.5, x=x.ptr, h=h.ptr, ld_h=ldh)
    call(ctx, "m40llm_ext_embed_tokens_async", C.byref(e), 1)
    want = od.embedding(tok, pos, ld.bf16_to_f32(E).astype(np.float64), 3.5, ld.bf16_to_f32(P).astype(np.float64))
    close_to(x.download(np.float32, (rows, width)), want, "float32")
    got = from_act(unpack_tiles(h.download(act_type(dtype), ((rows + 15) // 16 * 16 * ldh,)), rows, ldh), dtype)
    close_to(got[:, :width], want, dtype)
    assert np.all(got[:, width:] == 0)


def norm_add(ctx, dtype, x, w, eps, mult, **kw):
    rows, width = x.shape
    ldh = up32(width)
    dx, h, hr = ctx.to_device(x.astype(np.float32)), ctx.to_device(filled((rows + 15) // 16 * 16 * ldh, dtype)), ctx.to_device(filled((rows, ldh), dtype))
    dw = ctx.to_device(w.astype(np.float32))
    n = NormAdd(act_dtype=ACT[dtype], rows=rows, width=width, eps=eps, mult=mult, x=dx.ptr, w=dw.ptr, h=h.ptr, h_rows=hr.ptr, ld_h=ldh, **kw)
    call(ctx, "m40llm_ext_norm_add_rows_async", C.byref(n), 1)
    got = dx.download(np.float32, (rows, width))
    packed = from_act(unpack_tiles(h.download(act_type(dtype), ((rows + 15) // 16 * 16 * ldh,)), rows, ldh), dtype)
    plain = from_act(hr.download(act_type(dtype), (rows, ldh)), dtype)
    assert np.array_equal(packed, plain) and np.all(plain[:, width:] == 0)
    close_to(plain[:, :width], got, dtype)
    return got


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows,width,planes", [(1, 8, 1), (3, 36, 2), (200, 1024, 1), (17, 4100, 3), (5, 8200, 2)])
def test_norm_on_the_output_then_add(ctx, rows, width, planes, dtype):
    rng, keep = np.random.default_rng(width), []
    x, w, y = rng.standard_normal((rows, width)), 1 + 0.3 * rng.standard_normal(width), rng.standard_normal((planes, rows, width)) * 0.02
    eps = 4e-4                     # of the size of the mean square: it counts
    got = norm_add(ctx, dtype, x, w, eps, 0.7, planes=dev(ctx, keep, y, np.float32), n_planes=planes, plane_stride=rows * width)
    close_to(got, x.astype(np.float32) + 0.7 * od.rms_norm(y.astype(np.float32).astype(np.float64).sum(axis=0), w, eps), "float32", factor=2)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows,width,top", [(1, 36, 1), (40, 256, 3), (7, 4100, 4)])
def test_expert_outputs_gathered_normed_and_added(ctx, rows, width, top, dtype):
    rng, keep = np.random.default_rng(width + top), []
    x, w, weight = rng.standard_normal((rows, width)), 1 + 0.3 * rng.standard_normal(width), rng.random((rows, top))
    slots, ldo = rows * top + 5, (width + 7) // 8 * 8
    out = np.zeros((slots, ldo))
    out[:, :width] = rng.standard_normal((slots, width))
    place = rng.permutation(slots)[:rows * top].reshape(rows, top).astype(np.uint32)
    place[rng.random((rows, top)) < 0.3] = INPUT
    got = norm_add(ctx, dtype, x, w, 1e-3, 0.5, expert_out=dev(ctx, keep, as_act(out, dtype)), ld_expert=ldo, place=u32(ctx, keep, place),
                   weight=dev(ctx, keep, weight, np.float32), top=top)
    y = np.zeros((rows, width))
    for r in range(rows):
        for j in range(top):
            y[r] += weight[r, j] * (x[r].astype(np.float32) if place[r, j] == INPUT else rounded(out, dtype)[place[r, j], :width])
    close_to(got, x.astype(np.float32) + 0.5 * od.rms_norm(y, w, 1e-3), "float32", factor=2)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows,cols", [(1, 8), (20, 150), (3, 2048), (130, 9000)])
def test_norm_times_gate(ctx, rows, cols, dtype):
    rng, keep = np.random.default_rng(cols), []
    y, w, z = rng.standard_normal((rows, cols)) * 0.03, 1 + 0.3 * rng.standard_normal(cols), rng.standard_normal((rows, cols + 4)) * 2
    ldo = up32(cols)
    out = ctx.to_device(filled((rows + 15) // 16 * 16 * ldo, dtype))
    call(ctx, "m40llm_ext_norm_gate_rows_async", dev(ctx, keep, y, np.float32), C.c_uint64(cols), dev(ctx, keep, w, np.float32), dev(ctx, keep, z, np.float32),
         C.c_uint64(cols + 4), rows, cols, C.c_float(1e-3), out.ptr, ldo, ACT[dtype], 1)
    got = from_act(unpack_tiles(out.download(act_type(dtype), ((rows + 15) // 16 * 16 * ldo,)), rows, ldo), dtype)
    close_to(got[:, :cols], od.rms_norm(y, w, 1e-3) * od.sigmoid(z[:, :cols]), dtype)
    assert np.all(got[:, cols:] == 0)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows", [1, 30, 129])
@pytest.mark.parametrize("plain,active", [(16, 32), (0, 96), (48, 320)])
def test_projection_with_silu_columns(ctx, dtype, rows, plain, active):
    rng = np.random.default_rng(rows + active)
    A, W = rng.standard_normal((rows, 100)), bf16w(rng, plain + active, 100, 3.0)
    R = (rows + 15) // 16 * 16
    out = gemm(ctx, dtype, SILU_KIND, A, W, out_f32=np.full((rows, max(plain, 4)), 7.0, np.float32), out_act=filled(R * active, dtype), ld_out=max(plain, 4),
               ld_act=active, plain_tiles=plain // 16)
    z = rounded(A, dtype) @ W.T.astype(np.float64)
    if plain:
        close_to(out["out_f32"], z[:, :plain], "float32", factor=2)
    close_to(from_act(unpack_tiles(out["out_act"], rows, active), dtype), od.silu(z[:, plain:]), dtype, factor=2)


def test_rms_norm_of_chosen_rows(ctx):
    rng, keep = np.random.default_rng(1), []
    x, w = rng.standard_normal((9, 100)) + 1.5, 1 + 0.3 * rng.standard_normal(100)
    pick = np.array([8, 0, 0, 3])
    out = ctx.to_device(filled(16 * 128, "float32"))
    call(ctx, "m40llm_ext_norm_rows_async", RMS, dev(ctx, keep, x, np.float32), None, 0, C.c_uint64(0), dev(ctx, keep, w, np.float32), u32(ctx, keep, pick), 4,
         100, C.c_float(1e-2), out.ptr, 128, 1, 1)
    close_to(unpack_tiles(out.download(np.float32, (16 * 128,)), 4, 128)[:, :100], od.rms_norm(x, w, 1e-2)[pick], "float32", factor=2)


# ---- routing and products per expert ------------------------------------------------------------------------------------------------
def route(ctx, z, correction, experts, top, job_rows):
    rows, all_ = z.shape
    ctx.lib.m40llm_ext_expert_slots.restype = ctx.lib.m40llm_ext_expert_max_jobs.restype = C.c_uint32
    slots, jobs = ctx.lib.m40llm_ext_expert_slots(rows, experts, top), ctx.lib.m40llm_ext_expert_max_jobs(rows, experts, top, job_rows)
    keep = []
    ids, weight, rows_of, place, job = (ctx.to_device(np.full(n, 77, t)) for n, t in ((rows * top, np.uint32), (rows * top, np.float32), (slots, np.uint32),
                                                                                      (rows * top, np.uint32), (4 + 4 * jobs, np.uint32)))
    r = Route(rows=rows, experts=experts, identity=all_ - experts, top=top, job_rows=job_rows, scale=1.0, logits=dev(ctx, keep, z, np.float32), ld_logits=all_,
              correction=dev(ctx, keep, correction, np.float32), ids=ids.ptr, weight=weight.ptr, rows_of=rows_of.ptr, place=place.ptr, jobs=job.ptr)
    call(ctx, "m40llm_ext_route_rows_async", C.byref(r), 1)
    return (ids.download(np.uint32, (rows, top)), weight.download(np.float32, (rows, top)), rows_of, place, job, slots, jobs, keep)


@pytest.mark.parametrize("rows", [1, 5, 64, 65, 700])
@pytest.mark.parametrize("experts,identity,top", [(1, 0, 1), (4, 2, 3), (8, 0, 8), (60, 4, 6), (100, 28, 5), (200, 0, 2), (1000, 24, 9)])
@pytest.mark.parametrize("job_rows", [16, 128])
def test_choice_of_experts_and_sorted_list(ctx, rows, experts, identity, top, job_rows):
    rng = np.random.default_rng(rows + experts)
    n = experts + identity
    z, corr = (rng.standard_normal((rows, n)) * 2).astype(np.float32), (0.05 * rng.standard_normal(n)).astype(np.float32)
    if experts == 200:
        z[:, :] = z[:, :1]             # all equal: the lowest indices
        corr[:] = 0
    ids, weight, d_rows, d_place, d_jobs, slots, max_jobs, _ = route(ctx, z, corr, experts, top, job_rows)
    h = z.astype(np.float64)
    want, w = od.route(h, np.eye(n), corr.astype(np.float64), top)
    assert np.array_equal(np.sort(ids, axis=1), np.sort(want, axis=1))
    full = np.exp(h - h.max(axis=1, keepdims=True))
    full /= full.sum(axis=1, keepdims=True)
    assert np.allclose(weight, np.take_along_axis(full, ids.astype(int), axis=1), rtol=3e-6)
    rows_of, place, jobs = d_rows.download(np.uint32, (slots,)), d_place.download(np.uint32, (rows, top)), d_jobs.download(np.uint32, (4 + 4 * max_jobs,))
    assert np.array_equal(place == INPUT, ids >= experts)
    r, j = np.nonzero(ids < experts)
    assert np.array_equal(rows_of[place[r, j]], r) and len(set(place[r, j].tolist())) == len(r)
    seen = 0
    count = np.bincount(ids[ids < experts], minlength=experts)
    for e, s, m, _ in jobs[4:4 + 4 * jobs[0]].reshape(-1, 4):
        assert 1 <= m <= job_rows and s % 16 == 0
        own = np.isin(place, np.arange(s, s + m))
        assert own.sum() == m and np.all(ids[own] == e) and np.all(np.diff(rows_of[s:s + m].astype(int)) > 0)
        seen += m
    assert seen == count.sum() and jobs[0] <= max_jobs and jobs[1] == ((count + 15) // 16 * 16).sum() <= slots
    assert rows_of[:jobs[1]].max(initial=0) < rows


@pytest.mark.parametrize("dtype,job_rows", [("float32", 16), ("float32", 64), ("bfloat16", 16), ("bfloat16", 32), ("bfloat16", 64), ("bfloat16", 128)])
@pytest.mark.parametrize("rows,experts,top,width,ff", [(1, 3, 2, 64, 40), (50, 4, 3, 100, 70), (300, 5, 2, 256, 130), (200, 1, 1, 96, 16)])
def test_products_per_expert(ctx, dtype, job_rows, rows, experts, top, width, ff):
    """Gate and up through gathered rows (or rows put in list order first), then down, for every slot; one expert more than rows can choose."""
    rng, keep = np.random.default_rng(rows + ff), []
    z = rng.standard_normal((rows, experts)).astype(np.float32)
    if experts > 1:
        z[:, 1] = -50                  # nobody takes it
    ids, weight, d_rows, d_place, d_jobs, slots, max_jobs, k2 = route(ctx, z, np.zeros(experts, np.float32), experts, min(top, max(experts - 1, 1)), job_rows)
    place = d_place.download(np.uint32, ids.shape)
    h = rng.standard_normal((rows, width)).astype(np.float32)
    D, F = up32(width), up32(ff)
    tiles, down_tiles, dt = (ff + 15) // 16, (width + 15) // 16, D // 32
    plain = np.zeros((rows, D), act_type(dtype))
    plain[:, :width] = as_act(h, dtype)
    wg, wu, wd = ([bf16w(rng, n, k, g) for _ in range(experts)] for n, k, g in ((ff, width, 3.0), (ff, width, 1.0), (width, ff, 1.0)))
    w_in, w_out = [], []
    for e in range(experts):
        W = np.zeros((2 * tiles * 16, width), np.float32)
        for i in range(ff):
            W[i // 16 * 32 + i % 16], W[i // 16 * 32 + 16 + i % 16] = wg[e][i], wu[e][i]
        w_in.append(pack_tiles(ld.f32_to_bf16(W)))
        w_out.append(pack_tiles(ld.f32_to_bf16(wd[e])))
    rows_of = d_rows.ptr
    a, extra = dev(ctx, keep, plain), dict(gather=rows_of)
    if job_rows == 128:
        packed = ctx.to_device(np.zeros(slots * D, np.uint16))
        call(ctx, "m40llm_ext_gather_rows_async", a, D, C.c_void_p(rows_of), d_jobs.ptr, slots, packed.ptr, 1)
        a, extra = packed.ptr, {}
    act, out = ctx.to_device(np.zeros(slots * F, act_type(dtype))), ctx.to_device(filled((slots, width), dtype))
    common = dict(act_dtype=ACT[dtype], rows=rows, batches=1, jobs=d_jobs.ptr, max_jobs=max_jobs, job_rows=job_rows)
    g = Gemm(epilogue=PROJECT, a=a, lda=D, w=dev(ctx, keep, np.concatenate(w_in)), n_tiles=2 * tiles, k_tiles=dt, w_batch=2 * tiles * dt * 512, activation=SILU,
             out_act=act.ptr, ld_act=F, **extra, **common)
    call(ctx, "m40llm_ext_packed_gemm_async", C.byref(g), 1)
    g = Gemm(epilogue=STORE_ACT, a=act.ptr, lda=F, w=dev(ctx, keep, np.concatenate(w_out)), n_tiles=down_tiles, k_tiles=F // 32,
             w_batch=down_tiles * (F // 32) * 512, out_act=out.ptr, ld_act=width, cols=width, **common)
    call(ctx, "m40llm_ext_packed_gemm_async", C.byref(g), 1)
    got = from_act(out.download(act_type(dtype), (slots, width)), dtype)
    hr = rounded(h, dtype)
    want = np.stack([od.silu(hr @ wg[e].T.astype(np.float64)) * (hr @ wu[e].T) for e in range(experts)])
    want = np.stack([rounded(want[e], dtype) @ wd[e].T.astype(np.float64) for e in range(experts)])
    r, j = np.nonzero(ids < experts)
    close_to(got[place[r, j]], want[ids[r, j], r], dtype, factor=2)


# ---- differential attention -------------------------------------------------------------------------------------------------------------
class Cache:
    """A shuffled page table for some slots and the pages of one layer."""

    def __init__(self, ctx, dtype, G, dim, vdim, slots, max_pages, seed=0):
        ctx.lib.m40llm_ext_pair_page_elements.restype = C.c_uint64
        self.n = ctx.lib.m40llm_ext_pair_page_elements(2, G, dim, vdim)
        self.max_pages = max_pages
        self.table = np.random.default_rng(seed).permutation(slots * max_pages).astype(np.uint32).reshape(slots, max_pages)
        self.d_table = ctx.to_device(self.table)
        self.pages = ctx.to_device(np.zeros(slots * max_pages * self.n, act_type(dtype)))


def split(ctx, dtype, cache, cfg, proj, slot, pos, back, weights, state, source=False):
    """One launch over rows; returns queries [rows][H][2][dim]."""
    H, G, dim, vdim, taps, eps = cfg
    keep, rows = [], len(proj)
    k0 = (2 * H * dim + 15) // 16 * 16
    v0 = k0 + (2 * G * dim + 15) // 16 * 16
    pad = up32(dim)
    q = ctx.to_device(filled((rows, H, 2, pad), dtype))
    s = Split(act_dtype=ACT[dtype], rows=rows, maps=2, heads=H, kv_heads=G, dim=dim, vdim=vdim, taps=taps, eps=eps, proj=dev(ctx, keep, proj, np.float32),
              ld_proj=proj.shape[1], k_offset=k0, v_offset=v0, conv_state=state.ptr, ld_state=proj.shape[1], queries=q.ptr, cache=None if source else cache.pages.ptr,
              row_slot=u32(ctx, keep, slot), row_pos=u32(ctx, keep, pos), row_back=u32(ctx, keep, back), page_table=cache.d_table.ptr, max_pages=cache.max_pages)
    for n in ("q", "k", "v"):
        if taps:
            setattr(s, n + "_conv", dev(ctx, keep, weights[n + ".conv"].T, np.float32))
        if n != "v":
            setattr(s, n + "_norm", dev(ctx, keep, weights[n + ".norm"], np.float32))
    call(ctx, "m40llm_ext_pair_split_append_async", C.byref(s), 1)
    # what longer portions leave behind
    starts = [i for i in range(rows) if back[i] == 0]
    portions = [(i, next((j for j in range(i + 1, rows) if back[j] == 0 or back[j] == LONE), rows) - i, slot[i], 0) for i in starts]
    if portions and taps > 1:
        call(ctx, "m40llm_ext_conv_state_async", s.proj, C.c_uint64(proj.shape[1]), proj.shape[1], taps, state.ptr, C.c_uint64(proj.shape[1]),
             u32(ctx, keep, portions), s.row_pos, len(portions), 1)
    return from_act(q.download(act_type(dtype), (rows, H, 2, pad)), dtype)


SIZES = [(4, 2, 64, 128, 3), (3, 1, 20, 37, 4), (2, 2, 12, 8, 2), (1, 1, 1, 1, 1), (2, 1, 128, 96, 5), (2, 1, 256, 256, 3), (2, 2, 32, 64, 0)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,dim,vdim,taps", SIZES)
@pytest.mark.parametrize("cuts", [[70], [1] * 12, [2, 1, 3, 1, 1, 64, 2, 2, 130, 1]])
def test_convolution_norms_and_cache_append(ctx, dtype, H, G, dim, vdim, taps, cuts):
    """Two sequences side by side, cut the same way; queries against the restatement here, keys and values through a one-token attention
    in the tests below and, exactly, by their places here."""
    rng = np.random.default_rng(dim + taps)
    n, eps = sum(cuts), 1e-2
    k0 = (2 * H * dim + 15) // 16 * 16
    v0 = k0 + (2 * G * dim + 15) // 16 * 16
    cols = (v0 + G * vdim + 3) // 4 * 4
    u = rng.standard_normal((2, n, cols)).astype(np.float32)
    W = {c + ".conv": rng.standard_normal((m, max(taps, 1))) for c, m in (("q", 2 * H * dim), ("k", 2 * G * dim), ("v", G * vdim))}
    W |= {c + ".norm": 1 + 0.3 * rng.standard_normal(dim) for c in "qk"}
    W = {k: v.astype(np.float32).astype(np.float64) for k, v in W.items()}
    cache = Cache(ctx, dtype, G, dim, vdim, 3, (n + 63) // 64)
    state = ctx.to_device(np.full((3, max(taps - 1, 1), cols), 99.0, np.float32))
    got, at = [[], []], 0
    for c in cuts:
        proj = np.concatenate([u[0, at:at + c], u[1, at:at + c]])
        back = [LONE] if c == 1 else list(range(c))
        q = split(ctx, dtype, cache, (H, G, dim, vdim, taps, eps), proj, [2] * c + [0] * c, 2 * list(range(at, at + c)), 2 * back, W, state)
        got[0].append(q[:c]); got[1].append(q[c:])
        at += c
    pages = from_act(cache.pages.download(act_type(dtype), (3 * cache.max_pages, G, cache.n // G)), dtype)
    for i, slot in ((0, 2), (1, 0)):
        def conv(name, a, m):
            x = u[i, :, a:a + m].astype(np.float64)
            return od.short_convolution(x, np.zeros((taps - 1, m)), W[name + ".conv"])[0] if taps else x
        q = od.unit_heads(conv("q", 0, 2 * H * dim), 2 * H, dim, W["q.norm"], eps).reshape(n, H, 2, dim)
        g = np.concatenate(got[i])
        close_to(g[..., :dim], q, dtype)
        assert np.all(g[..., dim:] == 0)
        k = od.unit_heads(conv("k", k0, 2 * G * dim), 2 * G, dim, W["k.norm"], eps).reshape(n, G, 2, dim)
        v = conv("v", v0, G * vdim).reshape(n, G, vdim)
        kt, vt = up32(dim) // 32, (vdim + 15) // 16
        for p in range(n):
            page, t = pages[cache.table[slot, p // 64]], p % 64
            keys = page[:, :8 * kt * 512].reshape(G, 2, 4, kt, 4, 16, 8)[:, :, t // 16, :, :, t % 16].reshape(G, 2, -1)
            r = t % 32
            vals = page[:, 8 * kt * 512:].reshape(G, vt, 2, 4, 16, 8)[:, :, t // 32, r % 16 // 4, :, r // 16 * 4 + r % 4].reshape(G, -1)
            close_to(keys[..., :dim], k[p], dtype, scale=np.abs(k).max())
            close_to(vals[:, :vdim], v[p], dtype, scale=np.abs(v).max())
            assert np.all(keys[..., dim:] == 0) and np.all(vals[:, vdim:] == 0)


def fill_cache(ctx, dtype, cache, G, dim, vdim, slot_kv):
    kt, vt = up32(dim) // 32, (vdim + 15) // 16
    pages = np.zeros((cache.table.size, G, cache.n // G), np.float32)
    for slot, (k, v) in slot_kv.items():
        for p in range(len(k)):
            page, t = pages[cache.table[slot, p // 64]], p % 64
            kk, vv = np.zeros((G, 2, kt * 32)), np.zeros((G, vt * 16))
            kk[..., :dim], vv[:, :vdim] = k[p], v[p]
            page[:, :8 * kt * 512].reshape(G, 2, 4, kt, 4, 16, 8)[:, :, t // 16, :, :, t % 16] = kk.reshape(G, 2, kt, 4, 8)
            r = t % 32
            page[:, 8 * kt * 512:].reshape(G, vt, 2, 4, 16, 8)[:, :, t // 32, r % 16 // 4, :, r // 16 * 4 + r % 4] = vv.reshape(G, vt, 16)
    cache.pages = ctx.to_device(as_act(pages, dtype))


def attend(ctx, dtype, cache, cfg, q, gate, slot, pos, portions, form, splits=1, tile_queries=0):
    H, G, dim, vdim, scale, lam, out_scale, eps = cfg
    keep, rows, pad = [], len(q), up32(dim)
    group = H // G
    qq = np.zeros((rows, H, 2, pad), np.float32)
    qq[..., :dim] = q
    size = 16 if form == 0 else tile_queries
    tiles = [(r * group + i, min(size, n * group - i)) for r, n in portions for i in range(0, n * group, size)]
    ctx.lib.m40llm_ext_pair_attention_partial_floats.restype = C.c_uint64
    floats = ctx.lib.m40llm_ext_pair_attention_partial_floats(2, rows, H, vdim, splits)
    partial = ctx.alloc(max(floats, 4) * 4)
    ldo = up32(H * vdim)
    out = ctx.to_device(filled((rows + 15) // 16 * 16 * ldo, dtype))
    a = Attn(act_dtype=ACT[dtype], maps=2, form=form, heads=H, kv_heads=G, dim=dim, vdim=vdim, scale=scale, out_scale=out_scale, eps=eps,
             queries=dev(ctx, keep, as_act(qq, dtype)), cache=cache.pages.ptr, gate=dev(ctx, keep, gate, np.float32), ld_gate=gate.shape[1],
             row_slot=u32(ctx, keep, slot), row_pos=u32(ctx, keep, pos), page_table=cache.d_table.ptr, max_pages=cache.max_pages, tiles=u32(ctx, keep, tiles),
             n_tiles=len(tiles), tile_queries=tile_queries, splits=splits, first_row=0, n_rows=rows, partial=partial.ptr, partial_floats=floats, out=out.ptr, ld_out=ldo)
    setattr(a, "lambda", lam)
    call(ctx, "m40llm_ext_pair_attention_async", C.byref(a), 1)
    return from_act(unpack_tiles(out.download(act_type(dtype), ((rows + 15) // 16 * 16 * ldo,)), rows, ldo), dtype)[:, :H * vdim].reshape(rows, H, vdim)


def attend_want(q, k, v, pos, gate, cfg):
    H, G, dim, vdim, scale, lam, out_scale, eps = cfg
    out = np.zeros((len(q), H, vdim))
    for a in range(H):
        g = a // (H // G)
        m = [od.softmax_attend(q[:, a, i], k[:, g, i], v[:, g], scale, pos) for i in (0, 1)]
        out[:, a] = od.join_maps(m[0], m[1], lam, 1 - out_scale, eps) * od.sigmoid(gate[:, a:a + 1])
    return out


FORMS = [("float32", 0, 1, 0), ("bfloat16", 0, 1, 0), ("bfloat16", 0, 3, 0), ("bfloat16", 0, 40, 0), ("bfloat16", 1, 1, 64), ("bfloat16", 1, 1, 128)]


@pytest.mark.parametrize("dtype,form,splits,tile", FORMS)
@pytest.mark.parametrize("H,G,dim,vdim", [(4, 2, 64, 128), (3, 1, 20, 37), (2, 2, 32, 64), (1, 1, 1, 1), (6, 1, 128, 96), (2, 1, 160, 144)])
def test_differential_attention_with_one_key_that_stands_out(ctx, dtype, form, splits, tile, H, G, dim, vdim):
    """Every query row looks for one key by its first map (far away, at page borders, itself, the first) and for another by its second: what it
    finds is that token's values, less lambda times the other's."""
    if form == 1:
        most = ctx.lib.m40llm_ext_pair_attention_tile_queries(0, 2, dim, vdim)
        if most < tile:
            pytest.skip("these sizes have no such tile")
    rng = np.random.default_rng(dim)
    cfg = (H, G, dim, vdim, 1.0, 0.6, 0.8, 1e-5)
    n, rows = 330, 150
    cache = Cache(ctx, dtype, G, dim, vdim, 3, 6)
    kv = {}
    for slot in (0, 2):
        k, v = rng.standard_normal((n, G, 2, dim)) * 0.1, rng.standard_normal((n, G, vdim))
        kv[slot] = (rounded(k, dtype), rounded(v, dtype))
    fill_cache(ctx, dtype, cache, G, dim, vdim, kv)
    portions = [(0, 100), (100, 1), (101, rows - 101)]
    slot = [2] * 100 + [0] + [2] * (rows - 101)
    pos = list(range(200, 300)) + [n - 1] + list(range(280, 280 + rows - 101))
    q = np.zeros((rows, H, 2, dim))
    for r in range(rows):
        for a in range(H):
            for m in (0, 1):
                far = [0, 63, 64, pos[r], max(pos[r] - 1, 0), 127, 128, int(rng.integers(0, pos[r] + 1))][(r + a + 3 * m) % 8]
                key = kv[slot[r]][0][far, a // (H // G), m]
                q[r, a, m] = key / (key @ key) * 25 if dim > 1 else key * 3
    q = rounded(q, dtype)
    gate = rng.standard_normal((rows, H + 1)).astype(np.float32)
    got = attend(ctx, dtype, cache, cfg, q, gate, slot, pos, portions, form, splits, tile)
    for first, m in portions:
        k, v = kv[slot[first]]
        want = attend_want(q[first:first + m], k, v, pos[first:first + m], gate[first:first + m].astype(np.float64), cfg)
        close_to(got[first:first + m], want, dtype, factor=3)


@pytest.mark.parametrize("dtype,form,splits,tile", FORMS)
def test_differential_attention_over_many_like_keys(ctx, dtype, form, splits, tile):
    """Flat scores: every key counts, the pages' sums have to be complete; the maps nearly cancel."""
    rng = np.random.default_rng(3)
    H, G, dim, vdim = 4, 2, 64, 128
    cfg = (H, G, dim, vdim, 0.125, 0.9, 1.0, 1e-6)
    n = 700
    cache = Cache(ctx, dtype, G, dim, vdim, 2, 11)
    k, v = rounded(rng.standard_normal((n, G, 2, dim)), dtype), rounded(rng.standard_normal((n, G, vdim)) + 0.5, dtype)
    fill_cache(ctx, dtype, cache, G, dim, vdim, {1: (k, v)})
    pos = np.arange(n - 70, n)
    q, gate = rounded(rng.standard_normal((70, H, 2, dim)), dtype), rng.standard_normal((70, H)).astype(np.float32)
    got = attend(ctx, dtype, cache, cfg, q, gate, [1] * 70, pos, [(0, 70)], form, splits, tile)
    close_to(got, attend_want(q, k, v, pos, gate.astype(np.float64), cfg), dtype, factor=4)


# ---- lightning attention ----------------------------------------------------------------------------------------------------------------
def lightning(ctx, dtype, H, dim, vdim, decay, q, k, v, state, portions, pos, chunked):
    """q, k, v [rows][H][..] of one pass; state: device buffer [slots][H][dim][v_pad]."""
    keep, rows, dp, vp = [], len(q), up32(dim), up32(vdim)
    cols = H * (2 * dp + vp)
    x = np.zeros((rows, cols), np.float32)
    x[:, :H * dp].reshape(rows, H, dp)[..., :dim] = q
    x[:, H * dp:2 * H * dp].reshape(rows, H, dp)[..., :dim] = k
    x[:, 2 * H * dp:].reshape(rows, H, vp)[..., :vdim] = v
    groups, base = [], []
    for i, (r, n, _, _) in enumerate(portions):
        base.append(len(groups))
        groups += [(i, g * 64) for g in range(r // 64, (r + n - 1) // 64 + 1)]
    ctx.lib.m40llm_ext_lightning_scratch_bytes.restype = C.c_uint64
    nb = ctx.lib.m40llm_ext_lightning_scratch_bytes(len(groups), H, dim, vdim)
    scratch, o = ctx.alloc(nb), ctx.to_device(np.full((rows, H * vdim), 55.0, np.float32))
    l = Light(act_dtype=ACT[dtype], chunked=int(chunked), heads=H, dim=dim, vdim=vdim, qkv=dev(ctx, keep, pack_tiles(as_act(x, dtype))), ld_qkv=cols,
              log2_decay=dev(ctx, keep, np.log2(decay), np.float32), decay=dev(ctx, keep, decay, np.float32), state=state.ptr, o=o.ptr, ld_o=H * vdim,
              portions=u32(ctx, keep, portions), chunk_base=u32(ctx, keep, base), chunks=u32(ctx, keep, groups), row_pos=u32(ctx, keep, pos), n_portions=len(portions),
              n_chunks=len(groups), scratch=scratch.ptr, scratch_bytes=nb)
    call(ctx, "m40llm_ext_lightning_async", C.byref(l), 1)
    return o.download(np.float32, (rows, H, vdim))


@pytest.mark.parametrize("dtype,chunked", [("float32", 0), ("bfloat16", 0), ("bfloat16", 1)])
@pytest.mark.parametrize("H,dim,vdim", [(4, 128, 128), (3, 20, 40), (1, 1, 1), (2, 64, 200), (2, 256, 96), (1, 256, 256)])
def test_lightning_recurrence(ctx, dtype, chunked, H, dim, vdim):
    """Two passes over three slots: a fresh portion on a slot with old contents, one that goes on, short ones between that share their 64-row
    groups; 32-bit accuracy of everything behind the operands in every form, from fast decay to none."""
    rng = np.random.default_rng(dim + vdim)
    decay = np.array([0.35, 0.9, 0.999, 1.0][-H:])
    S = rng.standard_normal((3, H, dim, vdim)).astype(np.float32)
    vp = up32(vdim)
    full = np.zeros((3, H, dim, vp), np.float32)
    full[..., :vdim] = S
    state = ctx.to_device(full)
    S = S.astype(np.float64)
    starts = {0: 0, 1: 7, 2: 500}           # slot 0 is fresh: its old contents must not count
    for portions in ([(0, 90, 0), (90, 2, 1), (92, 37, 2)], [(0, 3, 2), (3, 200, 1), (203, 1, 0)]):
        rows = sum(p[1] for p in portions)
        q, k, v = (rounded(rng.standard_normal((rows, H, n)) * (0.3 if n == dim else 1.0), dtype) for n in (dim, dim, vdim))
        pos = np.zeros(rows, np.uint32)
        want = np.zeros((rows, H, vdim))
        for r, n, s in portions:
            pos[r:r + n] = starts[s] + np.arange(n)
            want[r:r + n], S[s] = od.lightning_recurrence(q[r:r + n], k[r:r + n], v[r:r + n], decay, S[s] if starts[s] else np.zeros_like(S[s]))
            starts[s] += n
        got = lightning(ctx, dtype, H, dim, vdim, decay, q, k, v, state, [(r, n, s, 0) for r, n, s in portions], pos, chunked)
        tol = 1e-5 if not chunked else 6e-5                    # two bf16 parts: 16 bits
        for h in range(H):
            assert np.abs(got[:, h] - want[:, h]).max() < tol * np.abs(want[:, h]).max(), (portions, h)
        end = state.download(np.float32, (3, H, dim, vp))[..., :vdim]
        for h in range(H):
            assert np.abs(end[:, h] - S[:, h]).max() < tol * np.abs(S[:, h]).max(), (portions, h)


def test_kernels_refuse_what_they_do_not_serve(ctx):
    b = ctx.alloc(1 << 16)
    p = {n: b.ptr for n in ("queries", "cache", "gate", "row_slot", "row_pos", "page_table", "tiles", "out")}
    ok = dict(maps=2, heads=2, kv_heads=1, dim=32, vdim=32, scale=1.0, ld_out=64, n_rows=1, n_tiles=1, splits=1, max_pages=1, **p)
    for bad, rc in ((dict(kv_heads=3), -3), (dict(dim=300), -3), (dict(scale=0.0), -3), (dict(ld_out=32), -3), (dict(form=1, tile_queries=96), -3),
                    (dict(splits=300), -3), (dict(maps=3), -3), (dict(splits=2), -4), (dict(cache=None), -1)):
        call(ctx, "m40llm_ext_pair_attention_async", C.byref(Attn(**dict(ok, **bad))), 1, rc=rc)
    p = {n: b.ptr for n in ("qkv", "decay", "log2_decay", "state", "o", "portions", "row_pos")}
    ok = dict(heads=1, dim=32, vdim=32, ld_qkv=96, ld_o=32, n_portions=1, **p)
    for bad, rc in ((dict(dim=257), -3), (dict(ld_qkv=64), -3), (dict(n_portions=0), -3), (dict(chunked=1), -4), (dict(state=None), -1)):
        call(ctx, "m40llm_ext_lightning_async", C.byref(Light(**dict(ok, **bad))), 1, rc=rc)
    p = {n: b.ptr for n in ("logits", "correction", "ids", "weight", "rows_of", "place", "jobs")}
    ok = dict(rows=1, experts=4, top=2, job_rows=16, ld_logits=4, **p)
    for bad, rc in ((dict(top=5), -3), (dict(experts=1025, ld_logits=1025), -3), (dict(job_rows=20), -3), (dict(ld_logits=3), -3), (dict(ids=None), -1)):
        call(ctx, "m40llm_ext_route_rows_async", C.byref(Route(**dict(ok, **bad))), 1, rc=rc)
    g = dict(act_dtype=0, epilogue=STORE_ACT, a=b.ptr, lda=64, w=b.ptr, n_tiles=2, k_tiles=2, rows=4, batches=1, out_act=b.ptr, ld_act=32, cols=32, jobs=b.ptr,
             max_jobs=1, job_rows=16)
    for bad in (dict(job_rows=8), dict(max_jobs=0), dict(batches=2), dict(gather=b.ptr), dict(epilogue=PROJECT), dict(act_dtype=1, job_rows=128)):
        call(ctx, "m40llm_ext_packed_gemm_async", C.byref(Gemm(**dict(g, **bad))), 1, rc=-3)
