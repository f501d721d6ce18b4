"""HIP kernels of mixers with a state per request, of windowed attention and of
what surrounds them, against the plain implementations of the same ops on the
CPU (ops/ref.py), over sizes on and off the tiles."""

import pytest
import torch

from substratus_amd.models.layers import (GluSpec, MoESpec, QueryTemperature,
                                          RotarySpec)
from substratus_amd.ops import hybrid as ops
from test_hybrid_ops_gpu import BS, close, make_batch, on_gpu, rand

pytestmark = pytest.mark.gpu

F32, BF16 = torch.float32, torch.bfloat16
BOTH = pytest.mark.parametrize("dtype", [F32, BF16])
# (first position, tokens) per request: single tokens and portions, at the
# start and later
SPANS = [(0, 1), (40, 1), (0, 5), (1, 2), (2, 37), (0, 70), (33, 19)]
LONG = [(7, 1), (0, 330), (3, 2), (60, 260)]


def cuda(*ts):
    return [t.cuda() if isinstance(t, torch.Tensor) else t for t in ts]


# ---- row operations ---------------------------------------------------------

@BOTH
@pytest.mark.parametrize("rows,width", [(3, 96), (70, 77), (4, 1024),
                                        (2, 9000), (5, 2050)])
@pytest.mark.parametrize("what", ["first", "rows", "all", "picked", "none"])
@pytest.mark.parametrize("layer", [True, False])
def test_add_norm(rows, width, what, layer, dtype):
    x = None if what == "first" else rand(rows, width, seed=1) + 0.5
    w, b = 1 + rand(width, seed=2), rand(width, seed=3) if layer else None
    r = rand(rows, width, seed=4, dtype=dtype) if what in ("rows", "all") \
        else None
    picked = None
    if what in ("picked", "all"):
        at = torch.randperm(rows * 5)[:rows * 5].int().view(rows, 5)
        picked = ops.Picked(rand(rows * 5, width, seed=5, dtype=dtype), at,
                            rand(rows, 5, seed=6))
    emb = vec = None
    if what in ("first", "all"):
        tok = torch.arange(rows, dtype=torch.int32) * 3 % 11
        emb = (tok, rand(11, width, seed=7, dtype=dtype), 1.7)
        vec = rand(width, seed=8)
    xg = None if x is None else x.cuda()
    gx, gy = ops.add_norm(xg, *cuda(w, b), 1e-5, dtype,
                          None if r is None else r.cuda(),
                          picked and ops.Picked(*cuda(*picked)),
                          emb and tuple(cuda(*emb)),
                          None if vec is None else vec.cuda())
    wx, wy = ops.add_norm(x, w, b, 1e-5, dtype, r, picked, emb, vec)
    assert gy.dtype == dtype and (xg is None or gx is xg)
    close(gx, wx, F32)
    close(gy, wy, dtype)


@BOTH
@pytest.mark.parametrize("n,pad", [(64, 8), (77, 3), (2048, 16), (5000, 1)])
def test_joint_gate(n, pad, dtype):
    o, norm = rand(9, n, seed=1, dtype=dtype), 1 + rand(n, seed=2)
    buf = rand(9, n + pad, seed=3, dtype=dtype)
    want, got = torch.zeros(9, n + pad, dtype=dtype), \
        torch.zeros(9, n + pad, dtype=dtype, device="cuda")
    ops.joint_gate(o, norm, buf[:, pad:], 1e-3, want[:, :n])
    ops.joint_gate(o.cuda(), norm.cuda(), buf.cuda()[:, pad:], 1e-3,
                   got[:, :n])
    close(got, want, dtype)


@BOTH
@pytest.mark.parametrize("f,pad", [(64, 8), (37, 3), (5632, 0)])
@pytest.mark.parametrize("act", ["silu", "relu", "clamped"])
def test_glu(f, pad, act, dtype):
    x = rand(9, 2 * f + pad, seed=1, dtype=dtype, scale=3.0)
    want, got = torch.zeros(9, f + pad, dtype=dtype), \
        torch.zeros(9, f + pad, dtype=dtype, device="cuda")
    spec = GluSpec(act, 1.3)
    ops.glu(x[:, pad:], spec, want[:, pad:])
    ops.glu(x.cuda()[:, pad:], spec, got[:, pad:])
    close(got, want, dtype)


@BOTH
@pytest.mark.parametrize("shape", [(3, 101), (5, 512)])
def test_softcap(shape, dtype):
    x = rand(*shape, seed=1, dtype=dtype, scale=40.0)
    close(ops.softcap(x.cuda(), 30.0), ops.softcap(x.clone(), 30.0), dtype)


@BOTH
@pytest.mark.parametrize("rows", [1, 7, 300])
@pytest.mark.parametrize("k,n,at", [(16, 96, 0), (24, 40, 16), (7, 33, 5),
                                    (128, 512, 0), (256, 128, 8)])
def test_linear32(rows, k, n, at, dtype):
    x = rand(rows, k + at + 8, seed=1, dtype=dtype)
    w = rand(n, k, seed=2, dtype=dtype)
    got = ops.linear32(x.cuda()[:, at:at + k], w.cuda())
    assert got.dtype == F32
    close(got, ops.linear32(x[:, at:at + k], w), F32)


def test_rope_table_far_away():
    batch = make_batch([(3, 9), (100, 1)])
    batch.positions[-1] = 900000
    rot = RotarySpec(500.0, 12, True)
    want = ops.rope_table(batch, rot, rot.turns(), {})
    got = ops.rope_table(on_gpu(batch), rot, rot.turns("cuda"), {})
    close(got, want, F32)


# ---- mixtures of gated experts ----------------------------------------------

@BOTH
@pytest.mark.parametrize("rows", [1, 5, 90, 700])
@pytest.mark.parametrize("width,ff,act", [(64, 96, "clamped"), (77, 13, "relu"),
                                          (128, 64, "silu"),
                                          (64, 42, "clamped")])
def test_gated_experts(rows, width, ff, act, dtype):
    spec = MoESpec(7, 3, ff, glu=GluSpec(act, 0.8), over_chosen=True,
                   bias=True)
    y = rand(rows, width, seed=1, dtype=dtype)
    router = rand(7, width, seed=2, dtype=dtype)
    bias = rand(7, seed=3)
    up = rand(7, 2 * ff, width, seed=4, dtype=dtype, scale=width ** -0.5 * 2)
    down = rand(7, width, ff, seed=5, dtype=dtype, scale=ff ** -0.5)
    # scores are of the same rounded rows: choices agree but for ties

    def total(p):
        return (p.rows.float()[p.at.long()] *
                p.weights[:, :, None]).sum(1).cpu()
    want = total(ops.experts(y, router, up, down, spec, bias))
    got = total(ops.experts(*cuda(y, router, up, down), spec, bias.cuda()))
    close(got, want, dtype)


# ---- convolutions -----------------------------------------------------------

def conv_state(spans, taps, channels, dtype, seed):
    """Slots with rubbish where a sequence begins, zeros before its start."""
    s = rand(len(spans), taps - 1, channels, seed=seed, dtype=dtype)
    for i, (first, _) in enumerate(spans):
        if first:
            s[i, :max(taps - 1 - first, 0)] = 0
    return s


@BOTH
@pytest.mark.parametrize("taps", [1, 2, 3, 4, 7])
@pytest.mark.parametrize("channels,pad", [(96, 0), (37, 3), (64, 5)])
@pytest.mark.parametrize("bias,act", [(True, True), (False, False)])
def test_short_conv(taps, channels, pad, bias, act, dtype):
    batch = make_batch(SPANS)
    n = batch.tokens.shape[0]
    x = rand(n, channels + pad, seed=1, dtype=dtype)
    w = rand(channels, taps, seed=2)
    b = rand(channels, seed=3) if bias else None
    state = conv_state(SPANS, taps, channels, dtype, 4)
    sg = state.cuda()
    want = ops.short_conv(x[:, pad:], w, b, act, state, batch)
    got = ops.short_conv(x.cuda()[:, pad:], *cuda(w, b), act, sg,
                         on_gpu(batch))
    close(got, want, dtype)
    assert torch.equal(sg.cpu(), state)


@BOTH
@pytest.mark.parametrize("heads,kv,dim,turned", [(4, 4, 64, 16), (6, 2, 24, 24),
                                                 (3, 1, 9, 6), (2, 2, 10, 2)])
@pytest.mark.parametrize("taps,bias", [(4, True), (2, False), (6, True)])
def test_conv_rope(heads, kv, dim, turned, taps, bias, dtype):
    batch = make_batch(SPANS)
    n, rows = batch.tokens.shape[0], (heads + kv) * dim
    buf = rand(n, rows + 8, seed=1, dtype=dtype)
    w = rand(rows, taps, seed=2)
    b = rand(rows, seed=3) if bias else None
    state = conv_state(SPANS, taps, rows, dtype, 4)
    rot = RotarySpec(100.0, turned, True)
    kc, vc = (torch.zeros(64, kv, BS, dim, dtype=dtype) for _ in range(2))
    sg, kg, vg, gb = state.cuda(), kc.cuda(), vc.cuda(), on_gpu(batch)
    got = ops.conv_rope(buf.cuda(), *cuda(b, w), sg,
                        ops.rope_table(gb, rot, rot.turns("cuda"), {}), kg, vg,
                        gb)
    want = ops.conv_rope(buf, b, w, state,
                         ops.rope_table(batch, rot, rot.turns(), {}), kc, vc,
                         batch)
    for g, r in ((got, want), (kg, kc), (vg, vc)):
        close(g, r, dtype)
    assert torch.equal(sg.cpu(), state)


# ---- recurrences ------------------------------------------------------------

@BOTH
@pytest.mark.parametrize("spans", [SPANS, LONG], ids=["short", "long"])
@pytest.mark.parametrize("channels,n,b_at", [(96, 16, 16), (40, 3, 5),
                                             (130, 32, 8), (24, 100, 0)])
@pytest.mark.parametrize("recurrent", [False, True])
def test_selective_scan(spans, channels, n, b_at, recurrent, dtype):
    batch = make_batch(spans)
    rows = batch.tokens.shape[0]
    u = rand(rows, channels, seed=1, dtype=dtype)
    buf = rand(rows, channels + 16, seed=2, dtype=dtype)
    z, zb = rand(rows, channels, seed=3, scale=2.0), rand(channels, seed=4) - 3
    low = rand(rows, b_at + 2 * n + 8, seed=5, dtype=dtype)
    a, d = -rand(channels, n, seed=6).exp(), rand(channels, seed=7)
    state = rand(len(spans), channels, n, seed=8)
    sg = state.cuda()
    want = torch.zeros(rows, channels + 5, dtype=dtype)
    got = want.cuda()
    ops.selective_scan(u, buf[:, 16:], z, zb, low, b_at, a, d, state, batch,
                       want[:, :channels], recurrent)
    ops.selective_scan(*cuda(u, buf[:, 16:], z, zb, low), b_at, *cuda(a, d),
                       sg, on_gpu(batch), got[:, :channels], recurrent)
    close(got, want, dtype)
    close(sg, state, F32)


@BOTH
@pytest.mark.parametrize("spans", [SPANS, LONG], ids=["short", "long"])
@pytest.mark.parametrize("heads,dim,vdim", [(2, 32, 64), (3, 17, 20),
                                            (1, 128, 128), (2, 8, 5),
                                            (2, 256, 40)])
@pytest.mark.parametrize("recurrent", [False, True])
def test_lightning(spans, heads, dim, vdim, recurrent, dtype):
    batch = make_batch(spans)
    rows, n = batch.tokens.shape[0], heads * (2 * dim + vdim)
    x = rand(rows, (n + 7) // 8 * 8 + 8, seed=1, dtype=dtype)
    decay = torch.tensor([0.999, 0.05, 0.6][:heads])
    state = rand(len(spans), heads, dim, vdim, seed=2)
    sg = state.cuda()
    want = ops.lightning(x, decay, state, batch, recurrent)
    got = ops.lightning(x.cuda(), decay.cuda(), sg, on_gpu(batch), recurrent)
    close(got, want, dtype)
    assert float((sg.cpu() - state).abs().max() / state.abs().max()) < 1e-4


def delta_inputs(batch, heads, kv, dim, vdim, dtype, seed, fast=0.0):
    rows = batch.tokens.shape[0]
    nq = kv * dim
    qkv = rand(rows, 2 * nq + heads * vdim, seed=seed, dtype=dtype)
    z = rand(rows, heads * dim, seed=seed + 1, scale=2.0)
    zb = rand(heads * dim, seed=seed + 2) - 2 + fast
    rate = rand(heads, seed=seed + 3).exp()
    beta = rand(rows, heads + 3, seed=seed + 4, dtype=dtype, scale=2.0)
    norm = 1 + rand(vdim, seed=seed + 5)
    gate = rand(rows, heads * vdim, seed=seed + 6, dtype=dtype)
    return qkv, z, zb, rate, beta[:, 3:], norm, gate


@BOTH
@pytest.mark.parametrize("spans", [SPANS, LONG], ids=["short", "long"])
@pytest.mark.parametrize("heads,kv,dim,vdim", [
    (2, 2, 32, 64), (3, 1, 17, 20), (4, 2, 128, 128), (2, 2, 8, 5),
    (1, 1, 256, 40), (2, 1, 64, 256), (1, 1, 600, 300)])
@pytest.mark.parametrize("fast", [0.0, 8.0])
@pytest.mark.parametrize("recurrent", [False, True])
def test_delta(spans, heads, kv, dim, vdim, fast, recurrent, dtype):
    """fast: decays that leave nothing of a channel within a few tokens."""
    batch = make_batch(spans)
    args = delta_inputs(batch, heads, kv, dim, vdim, dtype, 1, fast)
    state = rand(len(spans), heads, dim, vdim, seed=9, scale=0.3)
    sg = state.cuda()
    rows = batch.tokens.shape[0]
    want = torch.zeros(rows, heads * vdim + 5, dtype=dtype)
    got = want.cuda()
    ops.delta(*args, state, batch, kv, 1e-5, 0.8, want[:, :heads * vdim],
              recurrent)
    ops.delta(*cuda(*args), sg, on_gpu(batch), kv, 1e-5, 0.8,
              got[:, :heads * vdim], recurrent)
    close(got, want, dtype)
    assert float((sg.cpu() - state).abs().max() / state.abs().max()) < 1e-4


def test_padded_rows_touch_no_state():
    batch = make_batch([(0, 1), (40, 1)])
    batch.state_slots[1] = -1
    gb = on_gpu(batch)
    x = rand(2, 3 * 32 + 8, seed=1, dtype=BF16).cuda()
    state = rand(2, 1, 32, 32, seed=2).cuda()
    before = state.clone()
    ops.lightning(x, torch.tensor([0.9]).cuda(), state, gb)
    assert torch.equal(state[1], before[1])
    args = cuda(*delta_inputs(batch, 1, 1, 32, 32, BF16, 1))
    ops.delta(*args, state, gb, 1, 1e-5, 1.0,
              torch.empty(2, 32, dtype=BF16, device="cuda"))
    assert torch.equal(state[1], before[1])
    conv = rand(2, 3, 32, seed=3, dtype=BF16).cuda()
    was = conv.clone()
    ops.short_conv(x[:, :32], rand(32, 4, seed=4).cuda(), None, True, conv, gb)
    assert torch.equal(conv[1], was[1])


# ---- windowed attention -----------------------------------------------------

@BOTH
@pytest.mark.parametrize("window,keep", [(40, 4), (16, 0), (1, 1), (17, 33),
                                         (300, 2), (70, 130)])
@pytest.mark.parametrize("heads,kv,d,cap", [(4, 4, 64, 30.0), (6, 2, 40, 0.0),
                                            (2, 1, 20, 5.0), (4, 1, 128, 2.0)])
@pytest.mark.parametrize("any_size", [False, True])
def test_window_attention(window, keep, heads, kv, d, cap, any_size, dtype):
    """Scores sharp enough that one key more or less shows; rows of out lie
    in wider ones."""
    spans = [(0, 1), (15, 1), (299, 1), (0, 5), (30, 2), (50, 150)]
    batch = make_batch(spans)
    n = batch.tokens.shape[0]
    q = rand(n, heads * d, seed=1, dtype=dtype, scale=2.0)
    kc, vc = (rand(64, kv, BS, d, seed=s, dtype=dtype) for s in (2, 3))
    sink = rand(heads, seed=4, scale=2.0)
    args = (batch, d ** -0.5, 0, any_size, window, keep, cap)
    want = torch.zeros(n, heads * d + 5, dtype=dtype)
    got = want.cuda()
    ops.attn_ctx(q, None, kc, vc, None, *args, sink, 0.6,
                 want[:, :heads * d])
    ops.attn_ctx(*cuda(q, None, kc, vc), None, on_gpu(batch), *args[1:],
                 sink.cuda(), 0.6, got[:, :heads * d])
    close(got, want, dtype)


@pytest.mark.parametrize("window,keep,cap,sink", [(0, 0, 0.0, True),
                                                  (200, 5, 20.0, True),
                                                  (0, 0, 20.0, False)])
def test_long_contexts_shared_by_workgroups(window, keep, cap, sink):
    batch = make_batch([(900, 1), (63, 1)])
    q = rand(2, 256, seed=1, dtype=BF16, scale=3.0)
    kc, vc = (rand(64, 2, BS, 128, seed=s, dtype=BF16) for s in (2, 3))
    s = rand(2, seed=4, scale=2.0) + 3 if sink else None
    args = (0.09, 0, False, window, keep, cap)
    want = ops.attn_ctx(q, None, kc, vc, None, batch, *args, s)
    got = ops.attn_ctx(*cuda(q, None, kc, vc), None, on_gpu(batch), *args,
                       s.cuda() if sink else None)
    close(got, want, BF16)


# ---- attention by sigmoids behind convolutions ------------------------------

@BOTH
@pytest.mark.parametrize("spans", [SPANS, LONG])
@pytest.mark.parametrize("heads,kv,d,dv,taps", [
    (4, 2, 64, 40, 4), (7, 1, 56, 72, 3), (2, 2, 9, 7, 2), (3, 3, 128, 256, 1),
    (2, 1, 20, 300, 5), (16, 16, 128, 128, 4)])
def test_conv_qkv(spans, heads, kv, d, dv, taps, dtype):
    batch = make_batch(spans)
    n, rows = batch.tokens.shape[0], (heads + kv) * d + kv * dv
    buf = rand(n, rows + 8, seed=1, dtype=dtype)
    bias, w = rand(rows, seed=2), rand(rows, taps, seed=3)
    state = conv_state(spans, taps, rows, dtype, 4)
    caches = [torch.zeros(64, kv, BS, s, dtype=dtype) for s in (d, dv)]
    sg, *cg = cuda(state, *caches)
    temp = QueryTemperature(0.6, 13)
    want = ops.conv_qkv(buf, bias, w, state, *caches, batch, temp, 1e-3)
    got = ops.conv_qkv(*cuda(buf, bias, w), sg, *cg, on_gpu(batch), temp,
                       1e-3)
    close(got, want, dtype)
    for a, b in zip(cg, caches):
        close(a, b, dtype)
    assert torch.equal(sg.cpu(), state)


@BOTH
@pytest.mark.parametrize("heads,kv,d,dv", [(4, 4, 64, 64), (6, 2, 40, 72),
                                           (3, 1, 20, 12), (8, 1, 128, 128),
                                           (2, 2, 192, 256)])
@pytest.mark.parametrize("any_size", [False, True])
@pytest.mark.parametrize("window,gated", [(0, False), (37, True)])
def test_sigmoid_attention(heads, kv, d, dv, any_size, window, gated, dtype):
    spans = [(0, 1), (15, 1), (899, 1), (0, 5), (30, 2), (50, 150)]
    batch = make_batch(spans, blocks=96)
    n = batch.tokens.shape[0]
    q = rand(n, heads * d, seed=1, dtype=dtype, scale=2.0)
    kc, vc = (rand(96, kv, BS, s, seed=s, dtype=dtype) for s in (d, dv))
    gate = rand(n, heads, seed=2, dtype=dtype) if gated else None
    r = rand(heads, seed=3).abs(), rand(heads, seed=4).abs()
    wb = rand(heads, seed=5) - 2

    def run(q, gate, kc, vc, batch, r1, r2, wb):
        return ops.attn_ctx(q, gate, kc, vc, None, batch, d ** -0.5,
                            any_size=any_size, window=window, mult=0.7,
                            falloff=(r1, r2), weight_bias=wb)
    want = run(q, gate, kc, vc, batch, *r, wb)
    got = run(*cuda(q, gate, kc, vc), on_gpu(batch), *cuda(*r, wb))
    close(got, want, dtype)


@BOTH
@pytest.mark.parametrize("any_size", [False, True])
def test_falloff_before_a_softmax(any_size, dtype):
    batch = make_batch([(0, 1), (700, 1), (0, 40), (90, 70)])
    n = batch.tokens.shape[0]
    q = rand(n, 2 * 64, seed=1, dtype=dtype, scale=2.0)
    kc, vc = (rand(64, 1, BS, 64, seed=s, dtype=dtype) for s in (2, 3))
    r = torch.tensor([0.3, 1.5]), torch.tensor([2.0, 0.1])
    want = ops.attn_ctx(q, None, kc, vc, None, batch, 0.125, falloff=r)
    got = ops.attn_ctx(*cuda(q, None, kc, vc), None, on_gpu(batch), 0.125,
                       any_size=any_size, falloff=tuple(cuda(*r)))
    close(got, want, dtype)
