"""HIP kernels of hybrid models against the plain implementations of the same
ops on the CPU in float32 (ops/ref.py), over sizes on and off the tiles."""

import pytest
import torch

from substratus_amd.ops import hybrid as ops
from substratus_amd.serve.batch import StepBatch

pytestmark = pytest.mark.gpu

BS = 16
TOL = {torch.float32: 2e-5, torch.bfloat16: 1.2e-2}


def rand(*shape, seed, dtype=torch.float32, scale=1.0):
    g = torch.Generator().manual_seed(seed)
    return (torch.randn(*shape, generator=g) * scale).to(dtype)


def close(got, want, dtype, what=""):
    got, want = got.float().cpu(), want.float().cpu()
    assert torch.isfinite(got).all(), what
    err = float((got - want).abs().max() / want.abs().max().clamp(min=1e-6))
    assert err < TOL[dtype], (what, err)


def on_gpu(batch):
    return StepBatch(**{
        k: v.cuda() if isinstance(v, torch.Tensor) else v
        for k, v in vars(batch).items()})


def make_batch(spans, blocks=64, seed=0):
    """Requests with (first position, tokens) each, on shuffled pages."""
    perm = torch.randperm(blocks,
                          generator=torch.Generator().manual_seed(seed))
    entries, at = [], 0
    for i, (first, n) in enumerate(spans):
        need = (first + n + BS - 1) // BS
        entries.append(([1] * n, first, perm[at:at + need].tolist(), i, []))
        at += need
    assert at <= blocks
    return StepBatch.build(entries, BS, torch.device("cpu"))


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("rows,width", [(3, 96), (5, 100), (2, 77), (4, 1024),
                                        (1, 4096), (2, 9000), (1, 9001 // 2)])
def test_stream_norm(rows, width, dtype):
    d = rand(rows, width, seed=1, dtype=dtype)
    x = rand(rows, width, seed=2)
    wp, wn = rand(width, seed=3), rand(width, seed=4)
    xr = x.clone()
    want = ops.stream_norm(d, xr, wp, wn, 1.0, 1e-5, 0.7)
    xg = x.cuda()
    got = ops.stream_norm(d.cuda(), xg, wp.cuda(), wn.cuda(), 1.0, 1e-5, 0.7)
    close(got, want, dtype)
    close(xg, xr, torch.float32)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("width", [96, 77, 2048])
def test_embed_norm(width, dtype):
    table = rand(37, width, seed=5, dtype=dtype)
    w = rand(width, seed=6)
    tok = torch.tensor([0, 36, 5, 5], dtype=torch.int32)
    x0, y0 = ops.embed_norm(tok, table, w, 1.0, 1e-5)
    x1, y1 = ops.embed_norm(tok.cuda(), table.cuda(), w.cuda(), 1.0, 1e-5)
    assert torch.equal(x0, x1.cpu())
    close(y1, y0, dtype)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("f", [328, 37, 64])
def test_silu_mul(f, dtype):
    x = rand(5, 2 * f, seed=7, dtype=dtype, scale=3.0)
    close(ops.silu_mul(x.cuda()), ops.silu_mul(x), dtype)


# heads, kv heads, dim, vdim
SHAPES = [(5, 5, 96, 40), (4, 2, 64, 128), (6, 1, 32, 32), (8, 2, 128, 128),
          (3, 3, 40, 24), (2, 1, 20, 12), (5, 1, 256, 256), (2, 2, 112, 160)]


def attention_inputs(shape, batch, dtype, blocks, seed):
    h, g, d, dv = shape
    n = batch.tokens.shape[0]
    ld = (h * d + g * d + g * dv + h + 15) // 16 * 16
    buf = rand(n, ld, seed=seed, dtype=dtype)
    kc = rand(blocks, g, BS, d, seed=seed + 1, dtype=dtype)
    vc = rand(blocks, g, BS, dv, seed=seed + 2, dtype=dtype)
    return buf, kc, vc


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("shape", SHAPES)
@pytest.mark.parametrize("full", [True, False])
def test_qkv_prepare(shape, dtype, full):
    h, g, d, dv = shape
    batch = make_batch([(0, 5), (20, 1), (3, 19)])
    buf, kc, vc = attention_inputs(shape, batch, dtype, 64, 10)
    qw, kw = rand(h * d, seed=13), rand(g * d, seed=14)
    first = rand(batch.tokens.shape[0], g * dv, seed=15, dtype=dtype)
    lam = torch.tensor(0.3)
    norms = (qw, kw) if full else (None, None)
    blend = (first, lam) if full else (None, None)
    dev = [None if t is None else t.cuda() for t in norms + blend]
    bg, kg, vg = buf.cuda(), kc.cuda(), vc.cuda()
    ops.qkv_prepare(bg, h * d, *dev[:2], 1e-5, *dev[2:], kg, vg,
                    batch.slots.cuda())
    ops.qkv_prepare(buf, h * d, *norms, 1e-5, *blend, kc, vc, batch.slots)
    close(bg, buf, dtype, "q")
    close(kg, kc, dtype, "k")
    close(vg, vc, dtype, "v")


@pytest.mark.parametrize("dtype,any_size", [(torch.float32, False),
                                            (torch.bfloat16, False),
                                            (torch.bfloat16, True)])
@pytest.mark.parametrize("shape", SHAPES)
@pytest.mark.parametrize("chunk", [0, 24, 100])
def test_attention(shape, dtype, any_size, chunk):
    h, g, d, dv = shape
    batch = make_batch([(0, 1), (99, 1), (100, 1), (301, 1), (0, 2), (17, 70),
                        (290, 33), (0, 130)], blocks=96)
    buf, kc, vc = attention_inputs(shape, batch, dtype, 96, 20)
    # one sharp score per row, so that a wrong key shows
    buf[:, :h * d] *= 2.0
    bias = rand(h, 61, seed=23, scale=2.0)
    gate_at = h * d + g * d + g * dv
    args = (batch, d ** -0.5 * 1.3, chunk, any_size)
    want = ops.attn_ctx(buf[:, :h * d], buf[:, gate_at:gate_at + h], kc, vc,
                        bias, *args)
    bg = buf.cuda()
    got = ops.attn_ctx(bg[:, :h * d], bg[:, gate_at:gate_at + h], kc.cuda(),
                       vc.cuda(), bias.cuda(), on_gpu(batch), *args[1:])
    close(got, want, dtype)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_attention_plain(dtype):
    """Without bias and gate, long enough for several workgroups a context."""
    batch = make_batch([(1500, 1), (1023, 300)], blocks=192)
    buf, kc, vc = attention_inputs((4, 2, 64, 64), batch, dtype, 192, 30)
    want = ops.attn_ctx(buf[:, :256], None, kc, vc, None, batch, 0.125, 0)
    got = ops.attn_ctx(buf.cuda()[:, :256], None, kc.cuda(), vc.cuda(), None,
                       on_gpu(batch), 0.125, 0)
    close(got, want, dtype)


def gla_inputs(shape, batch, dtype, seed, z_shift=0.0):
    h, d, dv, r = shape
    n = batch.tokens.shape[0]
    ld = (2 * h * (d + dv) + r + 15) // 16 * 16
    x = rand(n, ld, seed=seed, dtype=dtype)
    a2 = rand(h * d, r, seed=seed + 1, scale=r ** -0.5)
    a2b = rand(h * d, seed=seed + 2) + z_shift
    norm = 1 + rand(dv, seed=seed + 3, scale=0.2)
    state = rand(8, h, d, dv, seed=seed + 4)
    return x, a2, a2b, norm, state


GLA_SHAPES = [(5, 48, 72, 16), (2, 64, 32, 33), (3, 128, 256, 16),
              (2, 40, 24, 8), (1, 20, 300, 5), (2, 256, 96, 16), (2, 17, 7, 3)]


@pytest.mark.parametrize("dtype,recurrent", [(torch.float32, False),
                                             (torch.bfloat16, False),
                                             (torch.bfloat16, True)])
@pytest.mark.parametrize("shape", GLA_SHAPES)
@pytest.mark.parametrize("tau,z_shift", [(16.0, 0.0), (1.0, -6.0)])
def test_gla(shape, dtype, recurrent, tau, z_shift):
    """tau 1 with a low gate decays by more than e^-60 within a few tokens."""
    batch = make_batch([(0, 1), (7, 1), (0, 2), (0, 31), (5, 33), (64, 100)])
    x, a2, a2b, norm, state = gla_inputs(shape, batch, dtype, 40, z_shift)
    dev = [t.cuda() for t in (x, a2, a2b, norm, state)]
    got = ops.gla(*dev, on_gpu(batch), tau, 1e-5, recurrent)
    want = ops.gla(x, a2, a2b, norm, state, batch, tau, 1e-5, recurrent)
    close(got, want, dtype, "out")
    close(dev[4], state, torch.float32 if dtype == torch.float32
          else torch.bfloat16, "state")
    # what enters the recurrence is 32-bit data: far closer than bf16
    err = float((dev[4].cpu() - state).abs().max() / state.abs().max())
    assert err < 1e-4, err


def test_gla_segments():
    """A long portion is cut into segments that run side by side."""
    batch = make_batch([(32, 1300), (0, 700)], blocks=160)
    x, a2, a2b, norm, state = gla_inputs((2, 64, 64, 16), batch,
                                         torch.bfloat16, 50, 3.0)
    dev = [t.cuda() for t in (x, a2, a2b, norm, state)]
    got = ops.gla(*dev, on_gpu(batch), 16.0, 1e-5)
    want = ops.gla(x, a2, a2b, norm, state, batch, 16.0, 1e-5)
    close(got, want, torch.bfloat16, "out")
    assert float((dev[4].cpu() - state).abs().max()
                 / state.abs().max()) < 1e-4


def test_gla_padded_rows_touch_no_state():
    batch = make_batch([(0, 1), (3, 1)])
    batch.state_slots[:] = -1
    x, a2, a2b, norm, state = gla_inputs((2, 64, 64, 16), batch,
                                         torch.bfloat16, 60)
    dev = [t.cuda() for t in (x, a2, a2b, norm, state)]
    got = ops.gla(*dev, on_gpu(batch), 16.0, 1e-5)
    want = ops.gla(x, a2, a2b, norm, state, batch, 16.0, 1e-5)
    close(got, want, torch.bfloat16)
    assert torch.equal(dev[4].cpu(), state)
