"""The building blocks of layers over residual streams one by one, through the C ABI: stream update, projections split into queries and cache,
attention of one map in its forms, choice within groups of experts, convolution with unit vectors, matrix memory and channel delta rule token by
token and chunk by chunk.  Inputs are made so that one key out of place, a lost state, a wrong group or a decay off by one token shows at once."""
import ctypes as C

import numpy as np
import pytest

pytestmark = pytest.mark.gpu

from natatar_common import sd  # noqa: E402
from oracle.latent_decoder import rotation  # noqa: E402
from oracle.output_norm_decoder import short_convolution, silu, softmax_attend  # noqa: E402
from pimosun_common import as_act, c_struct, close_to, from_act, ld, m40, unpack_tiles, up32  # noqa: E402
from test_gpu_layer_kernels import ACT, DTYPES, act_type, bf16w, call, gemm, rounded  # noqa: E402
from test_gpu_sublayer_kernels import LONE, dev, filled, u32  # noqa: E402

Update, Qkv, Attn, Route, DSplit, Memory, Delta = (c_struct("M40llm" + n) for n in ("StreamUpdate", "QkvSplit", "PairAttention", "Route", "DeltaSplit",
                                                                                   "MatrixMemory", "ChannelDelta"))
SPLIT_KIND = 9


@pytest.fixture(scope="module")
def ctx():
    yield m40.Context(0)


# ---- streams --------------------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows,width,streams,kind", [(1, 8, 1, "planes"), (5, 36, 2, "planes"), (130, 256, 3, "experts"), (17, 4100, 4, "experts"), (3, 8200, 4, "planes"),
                                                     (40, 100, 7, "planes"), (9, 64, 16, "experts"), (20, 96, 4, "none")])
@pytest.mark.parametrize("first", [False, True])
def test_streams_take_the_output_and_the_next_sublayer_reads_them(ctx, dtype, rows, width, streams, kind, first):
    rng, keep = np.random.default_rng(width + streams), []
    X = rng.standard_normal((streams, rows, width)).astype(np.float32)
    x0 = rng.standard_normal((rows, width)).astype(np.float32)
    mix, share, take = rng.standard_normal((streams, streams)), rng.standard_normal(streams), rng.standard_normal(streams)
    w, eps, mult = 1 + 0.3 * rng.standard_normal(width), 0.3, 0.6
    mix, share, take, w = (a.astype(np.float32) for a in (mix, share, take, w))
    old = np.stack([x0] * streams) if first else X
    y, kw = None, {}
    if kind == "planes":
        P = rng.standard_normal((3, rows, width)).astype(np.float32)
        y = P.astype(np.float64).sum(axis=0)
        kw = dict(planes=dev(ctx, keep, P), n_planes=3, plane_stride=rows * width)
    elif kind == "experts":
        top, slots, ldo = 3, rows * 3 + 5, (width + 7) // 8 * 8
        out = np.zeros((slots, ldo))
        out[:, :width] = rng.standard_normal((slots, width))
        place = rng.permutation(slots)[:rows * top].reshape(rows, top)
        weight = rng.random((rows, top)).astype(np.float32)
        y = np.einsum("rj,rjw->rw", weight.astype(np.float64), rounded(out, dtype)[place][..., :width])
        kw = dict(expert_out=dev(ctx, keep, as_act(out, dtype)), ld_expert=ldo, place=u32(ctx, keep, place), weight=dev(ctx, keep, weight), top=top)
    new = sd.write_streams(old.astype(np.float64), mix.astype(np.float64), share.astype(np.float64), y, mult) if y is not None else old.astype(np.float64)
    stride = (rows + 3) * width
    full = np.full((streams, rows + 3, width), 7.0, np.float32)
    full[:, :rows] = X
    ldh = up32(width)
    base = dict(act_dtype=ACT[dtype], width=width, streams=streams, eps=eps, mult=mult, stream_stride=stride, mix=dev(ctx, keep, mix), share=dev(ctx, keep, share), **kw)
    if first:
        base["x0"] = dev(ctx, keep, x0)
    dx, h, hr = ctx.to_device(full), ctx.to_device(filled((rows + 15) // 16 * 16 * ldh, dtype)), ctx.to_device(filled((rows, ldh), dtype))
    call(ctx, "m40llm_ext_stream_update_async", C.byref(Update(rows=rows, streams_x=dx.ptr, take=dev(ctx, keep, take), w=dev(ctx, keep, w), h=h.ptr, h_rows=hr.ptr,
                                                               ld_h=ldh, **base)), 1)
    got = dx.download(np.float32, full.shape)
    assert np.all(got[:, rows:] == 7.0)
    if y is None:
        assert np.array_equal(got[:, :rows], X)
    else:
        close_to(got[:, :rows], new, "float32", factor=2)
    plain = from_act(hr.download(act_type(dtype), (rows, ldh)), dtype)
    close_to(plain[:, :width], sd.rms_norm(sd.read_streams(new, take.astype(np.float64)), w, eps), dtype, factor=2)
    packed = from_act(unpack_tiles(h.download(act_type(dtype), ((rows + 15) // 16 * 16 * ldh,)), rows, ldh), dtype)
    assert np.array_equal(packed, plain) and np.all(plain[:, width:] == 0)
    # the sum of the streams, of all rows and of some at the end
    for pick in (None, np.array([rows - 1, 0, rows // 2])):
        dx, xo = ctx.to_device(full), ctx.to_device(np.full((rows, width), 9.0, np.float32))
        more = {} if pick is None else dict(row_index=u32(ctx, keep, pick), discard=1)
        call(ctx, "m40llm_ext_stream_update_async", C.byref(Update(rows=rows if pick is None else 3, streams_x=dx.ptr, x_out=xo.ptr, **base, **more)), 1)
        got, which = xo.download(np.float32, (rows, width)), np.arange(rows) if pick is None else pick
        close_to(got[which], new.sum(axis=0)[which], "float32", factor=3)
        assert np.all(np.delete(got, which, axis=0) == 9.0)
        if pick is not None or y is None:
            assert np.array_equal(dx.download(np.float32, full.shape), full)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows", [1, 30, 129])
def test_projection_with_columns_as_operand(ctx, dtype, rows):
    rng = np.random.default_rng(rows)
    A, W = rng.standard_normal((rows, 100)), bf16w(rng, 48 + 96, 100, 3.0)
    out = gemm(ctx, dtype, SPLIT_KIND, A, W, out_f32=np.full((rows, 48), 7.0, np.float32), out_act=filled((rows + 15) // 16 * 16 * 96, dtype), ld_out=48, ld_act=96,
               plain_tiles=3)
    z = rounded(A, dtype) @ W.T.astype(np.float64)
    close_to(out["out_f32"], z[:, :48], "float32", factor=2)
    close_to(from_act(unpack_tiles(out["out_act"], rows, 96), dtype), z[:, 48:], dtype, factor=2)


# ---- experts within groups ---------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("rows", [1, 40, 300])
@pytest.mark.parametrize("experts,count,keep,top,scale", [(8, 4, 3, 4, 2.0), (6, 3, 1, 2, 0.5), (64, 8, 2, 9, 1.0), (130, 13, 4, 6, 1.5), (512, 2, 1, 3, 1.0), (12, 12, 5, 5, 1.0), (5, 1, 1, 5, 3.0)])
def test_choice_within_the_best_groups(ctx, rows, experts, count, keep, top, scale):
    rng, bufs = np.random.default_rng(experts), []
    z = (rng.standard_normal((rows, experts)) * 2).astype(np.float32)
    z[0, :] = 0.25                    # all equal: the lowest indices
    # the two best experts overall, and one whose group does not make it in spite of a good second best
    if rows > 1 and count > keep > 0 and experts // count > 1:
        size = experts // count
        z[1] = np.repeat(np.arange(count)[::-1] * 0.5, size) - np.tile(np.arange(size) * 0.01, count)
        z[1, keep * size:(keep + 1) * size] = z[1, (keep - 1) * size] - 0.001
    slots, jobs = (getattr(ctx.lib, n)(rows, experts, top, *r) for n, r in (("m40llm_ext_expert_slots", ()), ("m40llm_ext_expert_max_jobs", (16,))))
    ids, weight, rows_of, place, job = (ctx.to_device(np.full(n, 77, t)) for n, t in ((rows * top, np.uint32), (rows * top, np.float32), (slots, np.uint32),
                                                                                      (rows * top, np.uint32), (4 + 4 * jobs, np.uint32)))
    call(ctx, "m40llm_ext_route_rows_async", C.byref(Route(rows=rows, experts=experts, top=top, job_rows=16, groups=count, keep=keep, scale=scale, ld_logits=experts,
                                                           logits=dev(ctx, bufs, z), ids=ids.ptr, weight=weight.ptr, rows_of=rows_of.ptr, place=place.ptr, jobs=job.ptr)), 1)
    want, w = sd.route(z.astype(np.float64), np.eye(experts), dict(top=top, scale=scale, groups=dict(count=count, keep=keep)))
    assert np.array_equal(ids.download(np.uint32, (rows, top)), want)
    assert np.allclose(weight.download(np.float32, (rows, top)), w, rtol=3e-6)


def test_routing_refuses_impossible_groups(ctx):
    b = ctx.alloc(1 << 16)
    p = {n: b.ptr for n in ("logits", "ids", "weight", "rows_of", "place", "jobs")}
    ok = dict(rows=1, experts=8, top=2, job_rows=16, ld_logits=8, scale=1.0, groups=4, keep=2, **p)
    for bad in (dict(groups=3), dict(keep=0), dict(keep=5), dict(keep=1, top=3)):
        call(ctx, "m40llm_ext_route_rows_async", C.byref(Route(**dict(ok, **bad))), 1, rc=-3)


# ---- attention of one map ------------------------------------------------------------------------------------------------------------------
class Cache:
    """A shuffled page table for some slots and the pages of one layer."""

    def __init__(self, ctx, dtype, G, dim, vdim, slots, max_pages, seed=0):
        ctx.lib.m40llm_ext_pair_page_elements.restype = C.c_uint64
        self.n = ctx.lib.m40llm_ext_pair_page_elements(1, G, dim, vdim)
        self.sizes, self.max_pages, self.dtype = (G, dim, vdim), max_pages, dtype
        self.table = np.random.default_rng(seed).permutation(slots * max_pages).astype(np.uint32).reshape(slots, max_pages)
        self.d_table = ctx.to_device(self.table)
        self.pages = ctx.to_device(np.zeros(slots * max_pages * self.n, act_type(dtype)))

    def views(self, page, t):
        """Where token t of a page [G][..] lies: keys [G][k_tiles][4][8], values [G][v_tiles][16]."""
        G, dim, vdim = self.sizes
        kt, vt, r = up32(dim) // 32, (vdim + 15) // 16, t % 32
        return (page[:, :4 * kt * 512].reshape(G, 4, kt, 4, 16, 8)[:, t // 16, :, :, t % 16],
                page[:, 4 * kt * 512:].reshape(G, vt, 2, 4, 16, 8)[:, :, t // 32, r % 16 // 4, :, r // 16 * 4 + r % 4])

    def fill(self, ctx, slot_kv):
        G, dim, vdim = self.sizes
        kt, vt = up32(dim) // 32, (vdim + 15) // 16
        pages = np.zeros((self.table.size, G, self.n // G), np.float32)
        for slot, (k, v) in slot_kv.items():
            for p in range(len(k)):
                kk, vv = np.zeros((G, kt * 32)), np.zeros((G, vt * 16))
                kk[:, :dim], vv[:, :vdim] = k[p], v[p]
                a, b = self.views(pages[self.table[slot, p // 64]], p % 64)
                a[:] = kk.reshape(G, kt, 4, 8)
                b[:] = vv.reshape(G, vt, 16)
        self.pages = ctx.to_device(as_act(pages, self.dtype))

    def read(self, slot, n):
        G, dim, vdim = self.sizes
        pages = from_act(self.pages.download(act_type(self.dtype), (self.table.size, G, self.n // G)), self.dtype)
        got = [self.views(pages[self.table[slot, p // 64]], p % 64) for p in range(n)]
        k, v = np.stack([a.reshape(G, -1) for a, _ in got]), np.stack([b.reshape(G, -1) for _, b in got])
        assert np.all(k[..., dim:] == 0) and np.all(v[..., vdim:] == 0)
        return k[..., :dim], v[..., :vdim]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,dim,vdim,rot", [(4, 2, 64, 128, 64), (3, 1, 21, 37, 10), (9, 3, 10, 12, 0), (2, 2, 12, 8, 4), (1, 1, 1, 1, 0), (2, 1, 256, 256, 64), (32, 4, 128, 96, 128)])
@pytest.mark.parametrize("options", ["plain", "biases", "norms", "keep", "first"])
def test_projections_become_queries_and_cache_entries(ctx, dtype, H, G, dim, vdim, rot, options):
    rng, keep = np.random.default_rng(dim + vdim), []
    eps, lam, n = 0.2, 0.3, 70
    slot = [2] * n + [0] * n
    pos = 2 * list(range(n))
    rows = len(slot)
    k0 = (H * dim + 15) // 16 * 16
    v0 = k0 + (G * dim + 15) // 16 * 16
    cols = (v0 + G * vdim + 3) // 4 * 4
    proj = rng.standard_normal((rows, cols)).astype(np.float32)
    proj[:, k0:k0 + G * dim] *= 0.4                    # the norms of queries and keys differ
    cache = Cache(ctx, dtype, G, dim, vdim, 3, 2)
    pad = up32(dim)
    dq, kept = ctx.to_device(filled((rows, H, pad), dtype)), ctx.to_device(np.full((rows, G * vdim), 5.0, np.float32))
    s = Qkv(act_dtype=ACT[dtype], rows=rows, heads=H, kv_heads=G, dim=dim, vdim=vdim, eps=eps, q_factor=-1.0 if options == "plain" else 1.0, proj=dev(ctx, keep, proj),
            ld_proj=cols, k_offset=k0, v_offset=v0, queries=dq.ptr, cache=cache.pages.ptr, row_slot=u32(ctx, keep, slot), row_pos=u32(ctx, keep, pos),
            page_table=cache.d_table.ptr, max_pages=cache.max_pages)
    parts = dict(q=proj[:, :H * dim].astype(np.float64), k=proj[:, k0:k0 + G * dim].astype(np.float64), v=proj[:, v0:v0 + G * vdim].astype(np.float64))
    if options in ("biases", "norms", "first"):
        for c in "qkv":
            b = rng.standard_normal(parts[c].shape[1]).astype(np.float32)
            parts[c] = parts[c] + b
            setattr(s, c + "_bias", dev(ctx, keep, b))
    if options in ("norms", "first"):
        for c in "qk":
            w = (1 + 0.3 * rng.standard_normal(parts[c].shape[1])).astype(np.float32)
            parts[c] = sd.rms_norm(parts[c], w, eps)
            setattr(s, c + "_norm", dev(ctx, keep, w))
    own = parts["v"]
    if options == "keep":
        s.keep_values, s.ld_values = kept.ptr, G * vdim
    if options == "first":
        f = rng.standard_normal(own.shape).astype(np.float32)
        s.first_values, s.ld_values = dev(ctx, keep, f), G * vdim
        setattr(s, "lambda", lam)
        parts["v"] = sd.mix_values(own, f, np.float64(np.float32(lam)))
    q, k, v = parts["q"].reshape(rows, H, dim), parts["k"].reshape(rows, G, dim), parts["v"].reshape(rows, G, vdim)
    if rot and options != "norms":
        spec = dict(base=300.0, dims=rot, scaling=dict(factor=4.0, original=64, fast=8.0, slow=0.5))
        f, mag = rotation(spec)
        a = np.array(pos)[:, None] * f[None, :]
        s.angles, s.rot_half = dev(ctx, keep, np.stack([np.cos(a) * mag, np.sin(a) * mag], axis=-1), np.float32), rot // 2
        q, k = sd.rotate(q, pos, spec), sd.rotate(k, pos, spec)
    call(ctx, "m40llm_ext_qkv_split_append_async", C.byref(s), 1)
    got = from_act(dq.download(act_type(dtype), (rows, H, pad)), dtype)
    close_to(got[..., :dim], q * s.q_factor, dtype)
    assert np.all(got[..., dim:] == 0)
    for i, sl in ((0, 2), (1, 0)):
        gk, gv = cache.read(sl, n)
        close_to(gk, k[i * n:(i + 1) * n], dtype)
        close_to(gv, v[i * n:(i + 1) * n], dtype)
    if options == "keep":
        close_to(kept.download(np.float32, own.shape), own, "float32")


def attend(ctx, dtype, cache, cfg, q, gate, slot, pos, portions, form, splits=1, tile_queries=0):
    H, G, dim, vdim, scale, out_scale = cfg
    keep, rows, pad = [], len(q), up32(dim)
    group = H // G
    qq = np.zeros((rows, H, pad), np.float32)
    qq[..., :dim] = q
    size = 16 if form == 0 else tile_queries
    tiles = [(r * group + i, min(size, n * group - i)) for r, n in portions for i in range(0, n * group, size)]
    ctx.lib.m40llm_ext_pair_attention_partial_floats.restype = C.c_uint64
    floats = ctx.lib.m40llm_ext_pair_attention_partial_floats(1, rows, H, vdim, splits)
    partial, ldo = ctx.alloc(max(floats, 4) * 4), up32(H * vdim)
    out = ctx.to_device(filled((rows + 15) // 16 * 16 * ldo, dtype))
    a = Attn(act_dtype=ACT[dtype], form=form, maps=1, heads=H, kv_heads=G, dim=dim, vdim=vdim, scale=scale, out_scale=out_scale,
             queries=dev(ctx, keep, as_act(qq, dtype)), cache=cache.pages.ptr, gate=None if gate is None else dev(ctx, keep, gate),
             ld_gate=0 if gate is None else gate.shape[1], row_slot=u32(ctx, keep, slot), row_pos=u32(ctx, keep, pos), page_table=cache.d_table.ptr,
             max_pages=cache.max_pages, tiles=u32(ctx, keep, tiles), n_tiles=len(tiles), tile_queries=tile_queries, splits=splits, first_row=0, n_rows=rows,
             partial=partial.ptr, partial_floats=floats, out=out.ptr, ld_out=ldo)
    call(ctx, "m40llm_ext_pair_attention_async", C.byref(a), 1)
    return from_act(unpack_tiles(out.download(act_type(dtype), ((rows + 15) // 16 * 16 * ldo,)), rows, ldo), dtype)[:, :H * vdim].reshape(rows, H, vdim)


def attend_want(q, k, v, pos, gate, cfg):
    H, G, dim, vdim, scale, out_scale = cfg
    out = np.stack([softmax_attend(q[:, a], k[:, a // (H // G)], v[:, a // (H // G)], scale, pos) for a in range(H)], axis=1) * out_scale
    return out if gate is None else out * sd.sigmoid(gate[:, :H * vdim].astype(np.float64)).reshape(out.shape)


FORMS = [("float32", 0, 1, 0), ("bfloat16", 0, 1, 0), ("bfloat16", 0, 3, 0), ("bfloat16", 0, 40, 0), ("bfloat16", 1, 1, 64), ("bfloat16", 1, 1, 128)]


@pytest.mark.parametrize("dtype,form,splits,tile", FORMS)
@pytest.mark.parametrize("H,G,dim,vdim", [(4, 2, 64, 64), (4, 2, 64, 128), (3, 1, 20, 37), (8, 2, 128, 128), (1, 1, 1, 1), (6, 1, 128, 96), (2, 1, 160, 144), (17, 1, 33, 16)])
@pytest.mark.parametrize("gated", [False, True])
def test_attention_with_one_key_that_stands_out(ctx, dtype, form, splits, tile, H, G, dim, vdim, gated):
    """Every query row looks for one key (far away, at page borders, itself, the one before, the first): what it finds is that token's values.
    The key just behind every row would win if it were seen."""
    if form == 1 and ctx.lib.m40llm_ext_pair_attention_tile_queries(0, 1, dim, vdim) < tile:
        pytest.skip("these sizes have no such tile")
    rng = np.random.default_rng(dim)
    cfg = (H, G, dim, vdim, 1.0, 0.8)
    n, rows = 330, 150
    cache = Cache(ctx, dtype, G, dim, vdim, 3, 6)
    kv = {}
    for slot in (0, 2):
        k, v = rng.standard_normal((n, G, dim)) * 0.1, rng.standard_normal((n, G, vdim))
        kv[slot] = (rounded(k, dtype), rounded(v, dtype))
    cache.fill(ctx, kv)
    portions = [(0, 100), (100, 1), (101, rows - 101)]
    slot = [2] * 100 + [0] + [2] * (rows - 101)
    pos = list(range(200, 300)) + [n - 1] + list(range(280, 280 + rows - 101))
    q = np.zeros((rows, H, dim))
    for r in range(rows):
        for a in range(H):
            far = [0, 63, 64, pos[r], pos[r] - 1, 127, 128, int(rng.integers(0, pos[r] + 1)), min(pos[r] + 1, n - 1)][(r + a) % 9]
            key = kv[slot[r]][0][far, a // (H // G)]
            q[r, a] = key / (key @ key) * 25 if dim > 1 else key * 3
    q = rounded(q, dtype)
    gate = rng.standard_normal((rows, H * vdim + (3 if dim == 20 else 4))).astype(np.float32) if gated else None
    got = attend(ctx, dtype, cache, cfg, q, gate, slot, pos, portions, form, splits, tile)
    for first, m in portions:
        k, v = kv[slot[first]]
        want = attend_want(q[first:first + m], k, v, pos[first:first + m], None if gate is None else gate[first:first + m], cfg)
        close_to(got[first:first + m], want, dtype, factor=3)


@pytest.mark.parametrize("dtype,form,splits,tile", FORMS)
def test_attention_over_many_like_keys(ctx, dtype, form, splits, tile):
    """Flat scores: every key counts, the pages' sums have to be complete."""
    rng = np.random.default_rng(3)
    H, G, dim, vdim, n = 4, 2, 64, 128, 700
    cfg = (H, G, dim, vdim, 0.125, 1.0)
    cache = Cache(ctx, dtype, G, dim, vdim, 2, 11)
    k, v = rounded(rng.standard_normal((n, G, dim)), dtype), rounded(rng.standard_normal((n, G, vdim)) + 0.5, dtype)
    cache.fill(ctx, {1: (k, v)})
    pos, q = np.arange(n - 70, n), rounded(rng.standard_normal((70, H, dim)), dtype)
    got = attend(ctx, dtype, cache, cfg, q, None, [1] * 70, pos, [(0, 70)], form, splits, tile)
    close_to(got, attend_want(q, k, v, pos, None, cfg), dtype, factor=2)


# ---- recurrences ---------------------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("H,G,dim,vdim,taps", [(4, 2, 64, 128, 4), (6, 3, 20, 37, 3), (2, 2, 12, 8, 2), (1, 1, 1, 1, 1), (2, 1, 128, 96, 5), (2, 1, 256, 256, 3), (3, 1, 33, 20, 4)])
@pytest.mark.parametrize("cuts", [[70], [1] * 12, [2, 1, 3, 1, 1, 64, 2, 2, 130, 1]])
def test_convolution_and_unit_vectors(ctx, H, G, dim, vdim, taps, cuts):
    """Two sequences side by side, cut the same way, on a ring with old contents."""
    rng = np.random.default_rng(dim + taps)
    n, sizes = sum(cuts), (("q", G * dim), ("k", G * dim), ("v", H * vdim))
    cols = 2 * G * dim + H * vdim
    ldp = (cols + 3) // 4 * 4
    u = rng.standard_normal((2, n, ldp)).astype(np.float32)
    u[:, 5] = 0                                       # a row whose unit vectors are nearly zero
    W = {c: rng.standard_normal((m, taps)).astype(np.float32) for c, m in sizes}
    state = ctx.to_device(np.full((3, max(taps - 1, 1), ldp), 99.0, np.float32))
    got, at = [[], []], 0
    for c in cuts:
        keep, proj = [], np.concatenate([u[0, at:at + c], u[1, at:at + c]])
        slot, pos, back = [2] * c + [0] * c, 2 * list(range(at, at + c)), 2 * ([LONE] if c == 1 else list(range(c)))
        out = ctx.to_device(np.full((2 * c, ldp), 55.0, np.float32))
        s = DSplit(rows=2 * c, heads=H, kv_heads=G, dim=dim, vdim=vdim, taps=taps, q_factor=0.7, proj=dev(ctx, keep, proj), ld_proj=ldp, conv_state=state.ptr, ld_state=ldp,
                   out=out.ptr, ld_out=ldp, row_slot=u32(ctx, keep, slot), row_pos=u32(ctx, keep, pos), row_back=u32(ctx, keep, back),
                   **{k + "_conv": dev(ctx, keep, w.T) for k, w in W.items()})
        call(ctx, "m40llm_ext_delta_split_async", C.byref(s), 1)
        if c > 1 and taps > 1:
            call(ctx, "m40llm_ext_conv_state_async", s.proj, C.c_uint64(ldp), cols, taps, state.ptr, C.c_uint64(ldp), u32(ctx, keep, [(0, c, 2, 0), (c, c, 0, 0)]), s.row_pos, 2, 1)
        g = out.download(np.float32, (2 * c, ldp))
        got[0].append(g[:c]); got[1].append(g[c:])
        at += c
    for i in (0, 1):
        g, a = np.concatenate(got[i]), 0
        for c, m in sizes:
            x = silu(short_convolution(u[i, :, a:a + m].astype(np.float64), np.zeros((taps - 1, m)), W[c].astype(np.float64))[0])
            if c != "v":
                x = sd.unit(x.reshape(n, G, dim)).reshape(n, m) * (0.7 if c == "q" else 1.0)
            close_to(g[:, a:a + m], x, "float32", factor=2)
            a += m


def chunk_tables(portions):
    groups, base = [], []
    for i, (r, n, _, _) in enumerate(portions):
        base.append(len(groups))
        groups += [(i, g * 64) for g in range(r // 64, (r + n - 1) // 64 + 1)]
    return base, groups


def run_recurrence(ctx, keep, name, struct, delta, chunked, portions, pos, out_cols, rows, dtype):
    base, groups = chunk_tables(portions)
    ctx.lib.m40llm_ext_memory_scratch_bytes.restype = C.c_uint64
    nb = ctx.lib.m40llm_ext_memory_scratch_bytes(int(delta), len(groups), struct.heads, struct.dim, struct.vdim)
    scratch = ctx.to_device(np.full(nb // 4, np.nan, np.float32))
    out = ctx.to_device(filled((rows + 15) // 16 * 16 * out_cols, dtype))
    struct.act_dtype, struct.chunked, struct.out, struct.ld_out = ACT[dtype], int(chunked), out.ptr, out_cols
    struct.portions, struct.chunk_base, struct.chunks, struct.row_pos = (u32(ctx, keep, a) for a in (portions, base, groups, pos))
    struct.n_portions, struct.n_chunks, struct.scratch, struct.scratch_bytes = len(portions), len(groups), scratch.ptr, nb
    call(ctx, name, C.byref(struct), 1)
    return from_act(unpack_tiles(out.download(act_type(dtype), ((rows + 15) // 16 * 16 * out_cols,)), rows, out_cols), dtype)


RUNS = [([(0, 90, 0), (90, 2, 1), (92, 37, 2)], "mixed"), ([(0, 3, 2), (3, 200, 1), (203, 1, 0)], "after"), ([(0, 64, 1), (64, 1, 2), (65, 150, 0)], "again")]
PATHS = [("float32", 0), ("bfloat16", 0), ("bfloat16", 1)]
SIZES = [(4, 128, 128), (3, 20, 40), (1, 1, 1), (2, 64, 200), (2, 256, 96), (1, 256, 256), (2, 130, 33), (3, 48, 64)]
# 32-bit accuracy of states in every form; outputs are rounded to the activation type
STATE_TOL = {0: 2e-5, 1: 6e-5}


def state_close(got, want, chunked, what):
    assert np.abs(got - want).max() < STATE_TOL[chunked] * max(np.abs(want).max(), 1e-3), (what, float(np.abs(got - want).max() / np.abs(want).max()))


@pytest.mark.parametrize("dtype,chunked", PATHS)
@pytest.mark.parametrize("H,dim,vdim", SIZES)
@pytest.mark.parametrize("gates", ["long", "short", "large"])
def test_matrix_memory(ctx, dtype, chunked, H, dim, vdim, gates):
    """Passes over three slots: a fresh portion on a slot with old contents, ones that go on, short ones that share their 64-row groups; memories
    that last for hundreds of tokens, that are lost within a few, and gates at their caps, whose running maximum jumps."""
    rng = np.random.default_rng(dim + vdim)
    cap, eps, factor = 7.0, 0.3, 0.6              # eps: the normalizer shows through the norm
    S = rng.standard_normal((3, H, dim, vdim)).astype(np.float32).astype(np.float64)
    N = rng.standard_normal((3, H, dim)).astype(np.float32).astype(np.float64)
    M = rng.uniform(0, 2, (3, H)).astype(np.float32).astype(np.float64)
    v4, d4 = (vdim + 3) // 4 * 4, (dim + 3) // 4 * 4
    ctx.lib.m40llm_ext_matrix_memory_state_floats.restype = C.c_uint64
    assert ctx.lib.m40llm_ext_matrix_memory_state_floats(dim, vdim) == dim * v4 + d4 + 4
    full = np.zeros((3, H, dim * v4 + d4 + 4), np.float32)
    full[..., :dim * v4].reshape(3, H, dim, v4)[..., :vdim] = S
    full[..., dim * v4:dim * v4 + dim], full[..., dim * v4 + d4] = N, M
    state = ctx.to_device(full)
    bias = [b.astype(np.float32) for b in ({"long": (-1.0, 6.0), "short": (0.0, -1.0), "large": (0.0, 0.0)}[gates] + rng.standard_normal((H, 2)) * 0.3).T]
    gain = {"long": 0.5, "short": 1.0, "large": 12.0}[gates]
    norm = (1 + 0.3 * rng.standard_normal(H * vdim)).astype(np.float32)
    starts = {0: 0, 1: 7, 2: 500}           # slot 0 is fresh: its old contents must not count
    for portions, what in RUNS:
        keep, rows, at, col = [], sum(p[1] for p in portions), 0, {}
        for c, m in (("q", H * dim), ("k", H * dim), ("v", H * vdim), ("g", H * vdim), ("i", H), ("f", H)):
            col[c] = at + (3 if dim == 20 else 4)     # offsets that allow wide loads, and that do not
            at = col[c] + (m + 3) // 4 * 4
        proj = rng.standard_normal((rows, at)).astype(np.float32)
        for c in "if":
            proj[:, col[c]:col[c] + H] *= gain
        p = {c: proj[:, col[c]:col[c] + m].astype(np.float64) for c, m in (("q", H * dim), ("k", H * dim), ("v", H * vdim), ("g", H * vdim), ("i", H), ("f", H))}
        i, f = sd.soft_cap(p["i"] + bias[0], cap), sd.log_sigmoid(sd.soft_cap(p["f"] + bias[1], cap))
        pos, want = np.zeros(rows, np.uint32), np.zeros((rows, H, vdim))
        for r, n, s in portions:
            pos[r:r + n] = starts[s] + np.arange(n)
            cut = slice(r, r + n)
            old = (S[s], N[s], M[s]) if starts[s] else (S[s] * 0, N[s] * 0, M[s] * 0)
            want[cut], S[s], N[s], M[s] = sd.memory_recurrence(p["q"][cut].reshape(n, H, dim) * dim ** -0.5, p["k"][cut].reshape(n, H, dim), p["v"][cut].reshape(n, H, vdim),
                                                               i[cut], f[cut], *old)
            starts[s] += n
        want = factor * sd.head_norm(want, eps).reshape(rows, H * vdim) * norm * sd.sigmoid(p["g"])
        m = Memory(heads=H, dim=dim, vdim=vdim, cap=cap, q_factor=dim ** -0.5, eps=eps, out_factor=factor, proj=dev(ctx, keep, proj), ld_proj=at, i_bias=dev(ctx, keep, bias[0]),
                   f_bias=dev(ctx, keep, bias[1]), norm=dev(ctx, keep, norm), state=state.ptr, out_col=32, **{c + "_col": col[c] for c in "qkvgif"})
        got = run_recurrence(ctx, keep, "m40llm_ext_matrix_memory_async", m, False, chunked, [(r, n, s, 0) for r, n, s in portions], pos, 32 + up32(H * vdim), rows, dtype)
        close_to(got[:, 32:32 + H * vdim], want, dtype, factor=20 if dtype == "float32" else 1)
        end = state.download(np.float32, full.shape)
        state_close(end[..., :dim * v4].reshape(3, H, dim, v4)[..., :vdim], S, chunked, (what, "S"))
        state_close(end[..., dim * v4:dim * v4 + dim], N, chunked, (what, "n"))
        state_close(end[..., dim * v4 + d4], M, chunked, (what, "m"))


@pytest.mark.parametrize("dtype,chunked", PATHS)
@pytest.mark.parametrize("H,dim,vdim", SIZES)
@pytest.mark.parametrize("keys", ["long", "short", "alike"])
def test_channel_delta_rule(ctx, dtype, chunked, H, dim, vdim, keys):
    """As above, with decays from none to a channel that is lost at once, and with keys that are nearly the same for many tokens, so that every write
    depends on the ones before it."""
    rng = np.random.default_rng(dim + vdim)
    G = 1 if H == 3 else H
    eps, factor = 1e-4, 1.3
    v4 = (vdim + 3) // 4 * 4
    S = rng.standard_normal((3, H, dim, vdim)).astype(np.float32).astype(np.float64)
    full = np.zeros((3, H, dim, v4), np.float32)
    full[..., :vdim] = S
    state = ctx.to_device(full)
    A_log = rng.uniform(-1.0, 1.0, H).astype(np.float32)
    dt = ({"long": -6.0, "short": 0.0, "alike": -4.0}[keys] + rng.standard_normal((H, dim)) * 2).astype(np.float32)
    dt[0, 0] = 30.0 if keys == "short" else dt[0, 0]          # a channel that keeps nothing
    norm = (1 + 0.3 * rng.standard_normal(vdim)).astype(np.float32)
    starts = {0: 0, 1: 7, 2: 500}
    share = np.arange(H) // (H // G)
    for portions, what in RUNS:
        keep, rows = [], sum(p[1] for p in portions)
        q, k = (sd.unit(rng.standard_normal((rows, G, dim)) * (0.2 if keys == "alike" else 1.0) + (1.0 if keys == "alike" else 0.0)) for _ in range(2))
        v = rng.standard_normal((rows, H, vdim))
        qkv = np.concatenate([a.reshape(rows, -1) for a in (q * 0.5, k, v)], axis=1).astype(np.float32)
        low = rng.standard_normal((rows, H * dim + 4 + H * vdim + 1)).astype(np.float32)
        beta = (rng.standard_normal((rows, H + 2)) * 2 + 2).astype(np.float32)
        q, k, v = (a.reshape(rows, -1, d).astype(np.float64) for a, d in zip(np.split(qkv, [G * dim, 2 * G * dim], axis=1), (dim, dim, vdim)))
        g = sd.channel_decay(low[:, :H * dim].reshape(rows, H, dim).astype(np.float64), A_log.astype(np.float64), dt.astype(np.float64))
        z, b = low[:, H * dim + 4:H * dim + 4 + H * vdim].astype(np.float64), sd.sigmoid(beta[:, 1:1 + H].astype(np.float64))
        pos, want = np.zeros(rows, np.uint32), np.zeros((rows, H, vdim))
        for r, n, s in portions:
            pos[r:r + n] = starts[s] + np.arange(n)
            cut = slice(r, r + n)
            want[cut], S[s] = sd.delta_recurrence(q[cut][:, share], k[cut][:, share], v[cut], g[cut], b[cut], S[s] if starts[s] else S[s] * 0)
            starts[s] += n
        want = factor * (sd.head_norm(want, eps) * norm).reshape(rows, H * vdim) * sd.sigmoid(z)
        d_beta = dev(ctx, keep, beta)
        m = Delta(heads=H, kv_heads=G, dim=dim, vdim=vdim, q_factor=1.0, eps=eps, out_factor=factor, qkv=dev(ctx, keep, qkv), ld_qkv=qkv.shape[1], low=dev(ctx, keep, low),
                  ld_low=low.shape[1], a_col=0, g_col=H * dim + 4, beta=d_beta + 4, ld_beta=H + 2, A_log=dev(ctx, keep, A_log), dt_bias=dev(ctx, keep, dt), norm=dev(ctx, keep, norm),
                  state=state.ptr)
        got = run_recurrence(ctx, keep, "m40llm_ext_channel_delta_async", m, True, chunked, [(r, n, s, 0) for r, n, s in portions], pos, up32(H * vdim), rows, dtype)
        close_to(got[:, :H * vdim], want, dtype, factor=20 if dtype == "float32" else 1)
        state_close(state.download(np.float32, full.shape)[..., :vdim], S, chunked, what)


def test_kernels_refuse_what_they_do_not_serve(ctx):
    b = ctx.alloc(1 << 16)

    def refuses(name, struct, ok, cases):
        for bad, rc in cases:
            call(ctx, name, C.byref(struct(**dict(ok, **bad))), 1, rc=rc)
    p = {n: b.ptr for n in ("streams_x", "mix", "share", "take", "planes", "w", "h")}
    refuses("m40llm_ext_stream_update_async", Update, dict(rows=1, width=32, streams=2, n_planes=1, ld_h=32, **p),
            [(dict(streams=17), -3), (dict(streams=0), -3), (dict(ld_h=16), -3), (dict(mix=None), -4), (dict(h=None), -1), (dict(w=None), -1), (dict(row_index=b.ptr), -4)])
    p = {n: b.ptr for n in ("proj", "queries", "cache", "row_slot", "row_pos", "page_table")}
    refuses("m40llm_ext_qkv_split_append_async", Qkv, dict(rows=1, heads=2, kv_heads=1, dim=32, vdim=32, k_offset=64, v_offset=96, ld_proj=128, **p),
            [(dict(heads=3, kv_heads=2), -3), (dict(dim=257), -3), (dict(ld_proj=127), -3), (dict(k_offset=60), -3), (dict(q_norm=b.ptr), -4), (dict(angles=b.ptr, rot_half=20), -4),
             (dict(first_values=b.ptr, ld_values=8), -4), (dict(cache=None), -1)])
    p = {n: b.ptr for n in ("proj", "q_conv", "k_conv", "v_conv", "out", "row_slot", "row_pos", "row_back")}
    refuses("m40llm_ext_delta_split_async", DSplit, dict(rows=1, heads=2, kv_heads=1, dim=8, vdim=8, taps=1, ld_proj=32, ld_out=32, **p),
            [(dict(taps=0), -3), (dict(dim=300), -3), (dict(ld_out=31), -3), (dict(heads=3, kv_heads=2), -3), (dict(taps=2), -4), (dict(q_conv=None), -1)])
    p = {n: b.ptr for n in ("proj", "i_bias", "f_bias", "norm", "state", "out", "portions", "row_pos")}
    refuses("m40llm_ext_matrix_memory_async", Memory, dict(heads=1, dim=8, vdim=8, cap=1.0, ld_proj=64, ld_out=32, n_portions=1, **p),
            [(dict(dim=257), -3), (dict(cap=0.0), -3), (dict(v_col=60), -3), (dict(ld_out=16), -3), (dict(n_portions=0), -3), (dict(chunked=1), -4), (dict(state=None), -1)])
    p = {n: b.ptr for n in ("qkv", "low", "beta", "A_log", "dt_bias", "norm", "state", "out", "portions", "row_pos")}
    refuses("m40llm_ext_channel_delta_async", Delta, dict(heads=2, kv_heads=1, dim=8, vdim=8, ld_qkv=32, ld_low=32, ld_beta=2, ld_out=32, n_portions=1, **p),
            [(dict(vdim=257), -3), (dict(heads=3, kv_heads=2), -3), (dict(ld_qkv=31), -3), (dict(ld_low=15), -3), (dict(ld_beta=1), -3), (dict(chunked=1), -4), (dict(norm=None), -1)])
