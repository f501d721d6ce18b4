"""HIP kernels of latent attention, mixtures of experts and side inputs against
the plain implementations of the same ops on the CPU (ops/ref.py), over sizes
on and off the tiles."""

import pytest
import torch

from substratus_amd.models.layers import (LatentAttentionSpec, MoESpec,
                                          RotarySpec)
from substratus_amd.ops import hybrid as ops
from test_hybrid_ops_gpu import BS, close, make_batch, on_gpu, rand

pytestmark = pytest.mark.gpu

F32, BF16 = torch.float32, torch.bfloat16
BOTH = pytest.mark.parametrize("dtype", [F32, BF16])


@BOTH
@pytest.mark.parametrize("rows,width,picks", [(3, 96, 2), (70, 77, 5),
                                              (4, 1024, 1), (2, 9000, 8)])
@pytest.mark.parametrize("pre", [True, False])
def test_stream_norm_of_picked_rows(rows, width, picks, pre, dtype):
    pool = rand(rows * picks + 3, width, seed=1, dtype=dtype)
    at = torch.randperm(rows * picks + 3)[:rows * picks].int().view(rows, -1)
    wt = rand(rows, picks, seed=2)
    x, wp, wn = rand(rows, width, seed=3), rand(width, seed=4), \
        rand(width, seed=5)
    xr, xg = x.clone(), x.cuda()
    want = ops.stream_norm(ops.Picked(pool, at, wt), xr, wp,
                           wn if pre else None, 0.0, 1e-5, mult=0.4)
    got = ops.stream_norm(ops.Picked(pool.cuda(), at.cuda(), wt.cuda()), xg,
                          wp.cuda(), wn.cuda() if pre else None, 0.0, 1e-5,
                          mult=0.4)
    assert got.dtype == dtype
    close(got, want, dtype)
    close(xg, xr, F32)


@BOTH
def test_embedding_without_a_norm(dtype):
    table = rand(37, 77, seed=5, dtype=dtype)
    tok = torch.tensor([0, 36, 5], dtype=torch.int32)
    x, y = ops.embed_norm(tok.cuda(), table.cuda(), None, 0.0, 1e-5)
    assert torch.equal(y.cpu(), table[tok.long()])
    assert torch.equal(x.cpu(), table[tok.long()].float())


# heads, dim, rot_dim, vdim, rank
SHAPES = [(4, 32, 16, 32, 64), (3, 24, 8, 40, 56), (16, 128, 64, 128, 512),
          (20, 64, 32, 48, 200), (2, 20, 6, 12, 37), (1, 8, 2, 8, 16),
          (5, 192, 64, 256, 448), (33, 16, 16, 16, 128), (2, 40, 40, 24, 600)]


def spec_of(shape, turned=None, **kw):
    h, d, r, dv, rank = shape
    return LatentAttentionSpec(h, d, r, dv, rank, 1.3 * (d + r) ** -0.5,
                               RotarySpec(1000.0, turned or r), **kw)


@BOTH
@pytest.mark.parametrize("shape", SHAPES)
@pytest.mark.parametrize("own", [True, False])
def test_latent_prepare(shape, own, dtype):
    batch = make_batch([(0, 5), (20, 1), (3, 19), (90, 1)])
    batch.positions[batch.positions == 90] = 900000
    spec = spec_of(shape, shape[2] // 2 // 2 * 2 or 2)
    n = batch.tokens.shape[0]
    nq, row = spec.heads * (spec.dim + spec.rot_dim), spec.row
    buf = rand(n, nq + 8 + row, seed=1, dtype=dtype)
    cache = torch.zeros(64, 1, BS, row, dtype=dtype)
    norm = 1 + rand(spec.rank, seed=2) if own else None
    bg, cg = buf.cuda(), cache.cuda()
    ops.latent_prepare(bg, spec, nq + 8 if own else -1,
                       norm.cuda() if own else None, 1e-4,
                       spec.rot.turns("cuda"), batch.positions.cuda(), cg,
                       batch.slots.cuda())
    ops.latent_prepare(buf, spec, nq + 8 if own else -1, norm, 1e-4,
                       spec.rot.turns(), batch.positions, cache, batch.slots)
    close(bg, buf, dtype, "q")
    close(cg, cache, dtype, "cache")


@BOTH
@pytest.mark.parametrize("rows", [1, 3, 17, 70])
@pytest.mark.parametrize("heads,k,n,tail", [
    (3, 32, 64, 16), (2, 128, 512, 64), (5, 20, 37, 6), (1, 8, 8, 0),
    (4, 200, 136, 8), (2, 512, 128, 0)])
@pytest.mark.parametrize("gated", [False, True])
def test_head_linear(rows, heads, k, n, tail, gated, dtype):
    x = rand(rows, heads * (k + tail) + 8, seed=1, dtype=dtype)
    w = rand(heads, n, k, seed=2, dtype=dtype, scale=k ** -0.5)
    gate = rand(rows, heads * n + 5, seed=3, dtype=dtype) if gated else None

    def run(x, w, g):
        v = x[:, :heads * (k + tail)].view(rows, heads, k + tail)
        return ops.head_linear(v, w, None if g is None else
                               g[:, 3:3 + heads * n], tail)
    want = run(x, w, gate)
    got = run(x.cuda(), w.cuda(), gate.cuda() if gated else None)
    close(got, want, dtype)
    if tail:
        assert torch.equal(got[..., n:].cpu(), want[..., n:])


def latent_inputs(spec, batch, dtype, blocks, seed, sharp=2.0):
    n = batch.tokens.shape[0]
    nq, ng = spec.heads * (spec.dim + spec.rot_dim), spec.heads * spec.vdim
    ld = (nq + ng + 15) // 16 * 16
    buf = rand(n, ld, seed=seed, dtype=dtype)
    buf[:, :nq] *= sharp          # one key stands out, so a wrong one shows
    cache = rand(blocks, 1, BS, spec.row, seed=seed + 1, dtype=dtype)
    w = rand(spec.heads * (spec.dim + spec.vdim), spec.rank, seed=seed + 2,
             dtype=dtype, scale=spec.rank ** -0.5)
    return buf, cache, w


def run_latent(spec, buf, cache, w, batch, expand=None, gated=True):
    nq, ng = spec.heads * (spec.dim + spec.rot_dim), spec.heads * spec.vdim
    uk_t = w[:spec.heads * spec.dim].view(spec.heads, spec.dim, spec.rank) \
        .transpose(1, 2).contiguous()
    return ops.latent_attn(buf[:, :nq], buf[:, nq:nq + ng] if gated else None,
                           cache, w, uk_t, batch, spec, {}, expand)


@pytest.mark.parametrize("dtype,expand", [(F32, None), (BF16, False),
                                          (BF16, True)])
@pytest.mark.parametrize("shape", SHAPES)
@pytest.mark.parametrize("gated", [True, False])
def test_latent_attention(shape, dtype, expand, gated):
    """Single tokens beside portions, from the first position and later ones,
    over several pages and steps; both ways to compute portions."""
    batch = make_batch([(0, 1), (99, 1), (128, 1), (301, 1), (0, 2), (17, 70),
                        (290, 33), (0, 130), (63, 2)], blocks=96)
    spec = spec_of(shape)
    args = latent_inputs(spec, batch, dtype, 96, 20)
    want = run_latent(spec, *args, batch, gated=gated)
    got = run_latent(spec, *(t.cuda() for t in args), on_gpu(batch), expand,
                     gated)
    close(got, want, dtype)


@pytest.mark.parametrize("first,n", [(1500, 1), (4000, 1), (1023, 3),
                                     (0, 1040)])
@pytest.mark.parametrize("expand", [True, False])
def test_latent_attention_long(first, n, expand):
    """Contexts that several workgroups share."""
    batch = make_batch([(first, n)], blocks=256)
    spec = spec_of((6, 32, 16, 32, 128))
    args = latent_inputs(spec, batch, BF16, 256, 30)
    want = run_latent(spec, *args, batch)
    got = run_latent(spec, *(t.cuda() for t in args), on_gpu(batch), expand)
    close(got, want, BF16)


@pytest.mark.parametrize("dtype,expand", [(F32, None), (BF16, False),
                                          (BF16, True)])
@pytest.mark.parametrize("shape", [(6, 32, 0, 32, 128), (3, 24, 0, 16, 40),
                                   (16, 128, 0, 128, 512), (2, 16, 8, 24, 64)])
@pytest.mark.parametrize("window", [1, 30, 64, 200, 1000])
def test_windowed_latent_attention(shape, window, dtype, expand):
    """Gates per head; a window alone, and beside a rotated key part."""
    batch = make_batch([(0, 1), (99, 1), (301, 1), (1023, 1), (0, 2), (17, 70),
                        (290, 33), (0, 330), (63, 2)], blocks=192)
    h, d, r, dv, rank = shape
    spec = LatentAttentionSpec(h, d, r, dv, rank, 1.3 * (d + r) ** -0.5, None,
                               head_gate=True, window=window)
    buf, cache, w = latent_inputs(spec, batch, dtype, 192, 40)
    uk_t = w[:h * d].view(h, d, rank).transpose(1, 2).contiguous()
    gate = rand(buf.shape[0], h + 1, seed=44, dtype=dtype)

    def run(buf, cache, w, uk_t, gate, batch, expand):
        return ops.latent_attn(buf[:, :h * (d + r)], gate[:, 1:], cache, w,
                               uk_t, batch, spec, {}, expand)
    want = run(buf, cache, w, uk_t, gate, batch, None)
    got = run(*(t.cuda() for t in (buf, cache, w, uk_t, gate)),
              on_gpu(batch), expand)
    close(got, want, dtype)


@pytest.mark.parametrize("z", [1, 5, 64, 65, 130, 1024])
@pytest.mark.parametrize("rows", [1, 7])
def test_moe_select_by_corrected_sigmoids(rows, z):
    from substratus_amd.ops import ref
    ext = ops._ext()
    corr = rand(z, seed=z) - 1.5
    for groups in (1, 2, 5, 13, 64):
        if z % groups:
            continue
        keep = (groups + 1) // 2
        for top in {1, min(6, keep * (z // groups))}:
            s = rand(rows, z, seed=z + groups, scale=2.0)
            ids = torch.empty(rows, top, dtype=torch.int32).cuda()
            wt = torch.empty(rows, top).cuda()
            ext.moe_select(ids, wt, torch.stack([s.cuda() * 0.25] * 4), groups,
                           keep, None, False, True, corr.cuda(), 2)
            ri, rw = ref.moe_select(s, top, groups, keep, False, True, corr, 2)
            assert torch.equal(ids.cpu(), ri), (groups, keep, top)
            assert torch.allclose(wt.cpu(), rw, rtol=1e-5), (groups, keep)


@pytest.mark.parametrize("z", [1, 5, 64, 65, 130, 1024])
@pytest.mark.parametrize("rows", [1, 7])
def test_moe_select(rows, z):
    from substratus_amd.ops import ref
    ext = ops._ext()
    for groups in (1, 2, 5, 8, 13, 64, 128):
        if z % groups:
            continue
        for keep in {1, (groups + 1) // 2, groups}:
            for top in {1, min(6, keep * (z // groups))}:
                s = rand(rows, z, seed=z + groups + keep, scale=2.0)
                ids = torch.empty(rows, top, dtype=torch.int32).cuda()
                wt = torch.empty(rows, top).cuda()
                ext.moe_select(ids, wt, torch.stack(
                    [s.cuda() * 0.25] * 4), groups, keep)
                ri, rw = ref.moe_select(s, top, groups, keep)
                assert torch.equal(ids.cpu(), ri), (groups, keep, top)
                assert torch.allclose(wt.cpu(), rw, rtol=1e-5), (groups, keep)


@pytest.mark.parametrize("n,top,experts,tile", [
    (1, 1, 1, 16), (5, 2, 8, 16), (300, 6, 32, 64), (9000, 3, 1000, 32),
    (64, 8, 5, 256)])
def test_moe_sort(n, top, experts, tile):
    ids = torch.randint(0, experts, (n, top), dtype=torch.int32,
                        generator=torch.Generator().manual_seed(n))
    if experts > 4:
        ids[ids == 3] = 0             # one without tokens
    packed = n * top
    i32 = dict(dtype=torch.int32, device="cuda")
    at = torch.empty(n, top, **i32)
    src = torch.empty(packed, **i32)
    start = torch.empty(experts + 1, **i32)
    tiles = torch.empty(1 + 2 * ((packed + tile - 1) // tile +
                                 min(experts, packed)), **i32)
    ops._ext().moe_sort(at, src, start, tiles, ids.cuda(), tile)
    at, src, start, tiles = (t.cpu().long() for t in (at, src, start, tiles))
    flat = ids.view(-1).long()
    counts = torch.bincount(flat, minlength=experts)
    assert torch.equal(start[1:], counts.cumsum(0)) and start[0] == 0
    where = at.view(-1)
    assert torch.equal(where.sort().values, torch.arange(packed))
    assert torch.equal(src[where], torch.arange(packed) // top)
    assert bool((where >= start[flat]).all() and
                (where < start[flat + 1]).all())
    want = [(e, r) for e in range(experts)
            for r in range(int(start[e]), int(start[e + 1]), tile)]
    assert int(tiles[0]) == len(want)
    assert tiles[1:1 + 2 * len(want)].view(-1, 2).tolist() == \
        [list(w) for w in want]


def combined(p):
    return (p.rows[p.at.long()].float() * p.weights[:, :, None]).sum(1)


@BOTH
@pytest.mark.parametrize("rows,width,experts", [
    (1, 4096, 32), (64, 4096, 33), (5, 77, 9), (300, 1024, 64), (20, 2048, 7)])
def test_router_scores(rows, width, experts, dtype):
    """32-bit sums, in shares of the width when there are few rows."""
    x = rand(rows, width, seed=1, dtype=dtype)
    w = rand(experts, width, seed=2, dtype=dtype, scale=width ** -0.5)
    got = ops._ext().router_scores(x.cuda(), w.cuda()).sum(0)
    close(got, x.double() @ w.double().T, F32)


@BOTH
@pytest.mark.parametrize("width,moe", [
    (96, MoESpec(16, 4, 64, 4, 3)), (64, MoESpec(3, 1, 40)),
    (51, MoESpec(6, 6, 37, 3, 3)), (256, MoESpec(4, 2, 320, 2, 1)),
    (128, MoESpec(1, 1, 64)), (192, MoESpec(70, 5, 72, 7, 2))])
@pytest.mark.parametrize("rows", [1, 5, 130, 1100])
def test_experts(rows, width, moe, dtype):
    """Rows per expert from none to as many as every tile size takes."""
    y = rand(rows, width, seed=1, dtype=dtype)
    router = rand(moe.experts, width, seed=2, dtype=dtype)
    up = rand(moe.experts, moe.ff, width, seed=3, dtype=dtype,
              scale=width ** -0.5)
    down = rand(moe.experts, width, moe.ff, seed=4, dtype=dtype,
                scale=moe.ff ** -0.5)
    want = ops.experts(y, router, up, down, moe)
    got = ops.experts(y.cuda(), router.cuda(), up.cuda(), down.cuda(), moe)
    close(combined(got), combined(want), dtype)


@pytest.mark.parametrize("tile", [16, 32, 64, 128, 256])
@pytest.mark.parametrize("k,n", [(64, 40), (192, 256), (640, 312)])
def test_expert_tiles(tile, k, n):
    """One product, packed rows in tiles of every size; experts with no rows,
    one row, and rows one off a tile's edge."""
    counts = [0, 1, tile, tile + 1, 2 * tile - 1, 0, 700]
    total, e = sum(counts), len(counts)
    g = torch.Generator().manual_seed(tile + k)
    ids = torch.repeat_interleave(torch.arange(e), torch.tensor(counts))
    ids = ids[torch.randperm(total, generator=g)].int()[:, None].contiguous()
    x = rand(total, k, seed=1, dtype=BF16)
    w = rand(e, n, k, seed=2, dtype=BF16, scale=k ** -0.5)
    i32 = dict(dtype=torch.int32, device="cuda")
    at, src = torch.empty(total, 1, **i32), torch.empty(total, **i32)
    start = torch.empty(e + 1, **i32)
    tiles = torch.empty(1 + 2 * ((total + tile - 1) // tile + e), **i32)
    ext = ops._ext()
    ext.moe_sort(at, src, start, tiles, ids.cuda(), tile)
    out = torch.full((total, n), 9.0, dtype=BF16, device="cuda")
    ext.expert_linear(out, x.cuda(), w.cuda(), src, start, tiles, tile, "gelu",
                      0.0)
    want = torch.empty(total, n)
    for i in range(e):
        r = ids[:, 0] == i
        want[r] = torch.nn.functional.gelu(x[r].float() @ w[i].float().T)
    close(out[at[:, 0].long()], want, BF16)


@BOTH
@pytest.mark.parametrize("rows,width,dim", [(1, 96, 16), (33, 77, 9),
                                            (300, 256, 128), (129, 192, 40)])
def test_side_gate(rows, width, dim, dtype):
    y = rand(rows, width, seed=1, dtype=dtype)
    w = rand(dim, width, seed=2, dtype=dtype, scale=width ** -0.5)
    table = rand(50, 3 * dim, seed=3, dtype=dtype)
    tok = torch.randint(0, 50, (rows,), dtype=torch.int32)
    want = ops.side_gate(y, w, tok, table, dim)
    got = ops.side_gate(y.cuda(), w.cuda(), tok.cuda(), table.cuda(), dim)
    close(got, want, dtype)
