"""Kernel microbenchmarks at llama2-7b decode shapes (run on MI355X).

Reports achieved bytes/s against the HBM ceiling (guide: 8 TB/s peak,
~6.3 TB/s achievable) for the decode hot kernels.
"""
import os
import sys
sys.path.insert(0, os.path.dirname(os.path.dirname(os.path.abspath(__file__))))

import argparse
import time

import torch

from substratus_amd import ops


def timeit(fn, iters=200, warmup=20):
    for _ in range(warmup):
        fn()
    torch.cuda.synchronize()
    t0 = time.time()
    for _ in range(iters):
        fn()
    torch.cuda.synchronize()
    return (time.time() - t0) / iters


def bench_attn(B=64, hq=32, hkv=32, d=128, ctx=512, bs=16):
    torch.manual_seed(0)
    nblk_per = (ctx + bs - 1) // bs
    nb = B * nblk_per + 1
    kc = torch.randn(nb, hkv, bs, d, device="cuda").bfloat16()
    vc = torch.randn_like(kc)
    bt = torch.arange(B * nblk_per, dtype=torch.int32,
                      device="cuda").reshape(B, nblk_per)
    q = torch.randn(B, hq, d, device="cuda").bfloat16()
    lens = torch.full((B,), ctx, dtype=torch.int32, device="cuda")
    scale = d ** -0.5
    dt = timeit(lambda: ops.paged_attn_decode(q, kc, vc, bt, lens, scale))
    kv_bytes = 2 * B * ctx * hkv * d * 2
    print(f"paged_attn_decode B={B} ctx={ctx} hq={hq} hkv={hkv} d={d}: "
          f"{dt*1e6:.1f} us, {kv_bytes/dt/1e12:.2f} TB/s")


def bench_rope(B=64, hq=32, hkv=32, d=128, bs=16):
    torch.manual_seed(0)
    nb = B * 4
    q = torch.randn(B, hq, d, device="cuda").bfloat16()
    k = torch.randn(B, hkv, d, device="cuda").bfloat16()
    v = torch.randn(B, hkv, d, device="cuda").bfloat16()
    pos = torch.full((B,), 500, dtype=torch.int32, device="cuda")
    slots = torch.arange(B, dtype=torch.int32, device="cuda")
    kc = torch.zeros(nb, hkv, bs, d, device="cuda").bfloat16()
    vc = torch.zeros_like(kc)
    dt = timeit(lambda: ops.rope_kv_append(q, k, v, pos, kc, vc, slots,
                                           10000.0))
    print(f"rope_kv_append B={B}: {dt*1e6:.1f} us")


def bench_norm(B=64, h=4096):
    x = torch.randn(B, h, device="cuda").bfloat16()
    r = torch.randn(B, h, device="cuda").bfloat16()
    w = torch.randn(h, device="cuda").bfloat16()
    dt = timeit(lambda: ops.rms_norm_residual(x, r, w, 1e-5))
    print(f"rms_norm_residual B={B} h={h}: {dt*1e6:.1f} us")


HBM = 8.0e12          # bytes/s
MFMA = 2.5e15         # dense bf16 flop/s


def report(name, dt, nbytes, flops=0.0):
    """Time beside the roofline: the larger of the HBM and matrix-core times
    of the work the op cannot avoid."""
    ideal = max(nbytes / HBM, flops / MFMA)
    print(f"{name:58s} {dt*1e6:9.1f} us  {nbytes/dt/1e12:5.2f} TB/s "
          f"{flops/dt/1e12:6.0f} TF/s  {100*ideal/dt:5.1f}% of roofline",
          flush=True)


def bench_hybrid():
    """Kernels of hybrid-layer models beside the like kernels of the uniform
    families, at equal sizes."""
    from substratus_amd.ops import hybrid as hy
    from substratus_amd.serve.batch import StepBatch
    torch.manual_seed(0)
    bf = dict(device="cuda", dtype=torch.bfloat16)

    def batch_of(n, first, tokens):
        need = (first + tokens + 15) // 16
        return StepBatch.build(
            [([1] * tokens, first, list(range(i * need, (i + 1) * need)), i,
              []) for i in range(n)], 16, torch.device("cuda"))

    for rows, w in ((64, 4096), (256, 4096), (16384, 4096)):
        x = torch.randn(rows, w, **bf)
        r = torch.randn(rows, w, **bf)
        wt = torch.randn(w, **bf)
        it = 200 if rows < 1000 else 50
        report(f"rms_norm_residual rows={rows} w={w}",
               timeit(lambda: ops.rms_norm_residual(x, r, wt, 1e-5), it),
               rows * w * 8)
        xf = torch.randn(rows, w, device="cuda")
        w32 = torch.randn(w, device="cuda")
        report(f"  stream_norm rows={rows} w={w}",
               timeit(lambda: hy.stream_norm(x, xf, w32, w32, 1.0, 1e-5), it),
               rows * w * 12)

    h, d = 32, 128
    for rows in (64, 256, 16384):
        nb = (rows + 15) // 16
        buf = torch.randn(rows, 3 * h * d + 32, **bf)
        kc = torch.zeros(nb, h, 16, d, **bf)
        vc = torch.zeros_like(kc)
        pos = torch.arange(rows, device="cuda", dtype=torch.int32)
        q, k, v = (buf[:, i * h * d:(i + 1) * h * d].view(rows, h, d)
                   for i in range(3))
        it = 200 if rows < 1000 else 50
        report(f"rope_kv_append rows={rows} {h}x{d}",
               timeit(lambda: ops.rope_kv_append(q, k, v, pos, kc, vc, pos,
                                                 1e4), it),
               rows * h * d * 2 * 7)
        w32 = torch.ones(h * d, device="cuda")
        vf = torch.randn(rows, h * d, **bf)
        lam = torch.tensor(0.5, device="cuda")
        report(f"  qkv_prepare rows={rows} {h}x{d}",
               timeit(lambda: hy.qkv_prepare(buf, h * d, w32, w32, 1e-5, vf,
                                             lam, kc, vc, pos), it),
               rows * h * d * 2 * 7)
        del buf, kc, vc, q, k, v, vf

    bias = torch.randn(h, 4096, device="cuda")
    for b, ctx, hq, hkv in ((8, 512, 32, 32), (64, 512, 32, 32),
                            (256, 512, 32, 32), (64, 2048, 32, 32),
                            (64, 2048, 32, 8)):
        nb = b * ctx // 16
        kc = torch.randn(nb, hkv, 16, d, **bf)
        vc = torch.randn_like(kc)
        q = torch.randn(b, hq * d, **bf)
        bt = torch.arange(nb, device="cuda", dtype=torch.int32).view(b, -1)
        lens = torch.full((b,), ctx, device="cuda", dtype=torch.int32)
        nbytes = 2 * b * ctx * hkv * d * 2
        it = 100
        report(f"paged_attn_decode b={b} ctx={ctx} {hq}/{hkv}x{d}",
               timeit(lambda: ops.paged_attn_decode(
                   q.view(b, hq, d), kc, vc, bt, lens, d ** -0.5), it),
               nbytes)
        sb = batch_of(b, ctx - 1, 1)
        gate = torch.randn(b, hq, **bf)
        report(f"  attn_ctx single b={b} ctx={ctx} {hq}/{hkv}x{d}",
               timeit(lambda: hy.attn_ctx(q, gate, kc, vc, bias, sb,
                                          d ** -0.5, 4096), it), nbytes)
        del kc, vc

    for b, s_ in ((32, 512), (8, 2048), (4, 4096)):
        t = b * s_
        q, k, v = (torch.randn(t, h, d, **bf) for _ in range(3))
        ss = torch.arange(0, t + 1, s_, dtype=torch.int32, device="cuda")
        flops = 4.0 * b * h * (s_ * (s_ + 1) / 2) * d
        nbytes = 4 * t * h * d * 2
        report(f"attn_v5 b={b} s={s_} {h}x{d}",
               timeit(lambda: ops.attn_prefill(q, k, v, ss, d ** -0.5), 20),
               nbytes, flops)
        sb = batch_of(b, 0, s_)
        kc = torch.randn(t // 16, h, 16, d, **bf)
        vc = torch.randn_like(kc)
        gate = torch.randn(t, h, **bf)
        q2 = q.view(t, h * d)
        report(f"  attn_ctx portions b={b} s={s_} {h}x{d}",
               timeit(lambda: hy.attn_ctx(q2, gate, kc, vc, bias, sb,
                                          d ** -0.5, 4096), 20),
               nbytes, flops)
        del q, k, v, kc, vc

    gh, gd, gv, r = 16, 128, 256, 16
    a2 = torch.randn(gh * gd, r, device="cuda") * 0.25
    ab = torch.randn(gh * gd, device="cuda")
    nw = torch.ones(gv, device="cuda")
    ld = 2 * gh * (gd + gv) + r
    for b in (8, 64, 256):
        state = torch.zeros(b, gh, gd, gv, device="cuda")
        x = torch.randn(b, ld, **bf)
        sb = batch_of(b, 100, 1)
        report(f"  gla single b={b} {gh}x{gd}x{gv}",
               timeit(lambda: hy.gla(x, a2, ab, nw, state, sb, 16.0, 1e-5),
                      100), state.numel() * 8 + x.numel() * 2)
    for b, s_ in ((32, 512), (8, 2048), (1, 8192)):
        t = b * s_
        state = torch.zeros(b, gh, gd, gv, device="cuda")
        x = torch.randn(t, ld, **bf)
        sb = batch_of(b, 0, s_)
        # two state products and, within chunks of 32, two score products
        flops = t * gh * (4.0 * gd * gv + 32.0 * (gd + gv))
        report(f"  gla portions b={b} s={s_} {gh}x{gd}x{gv}",
               timeit(lambda: hy.gla(x, a2, ab, nw, state, sb, 16.0, 1e-5),
                      20), x.numel() * 2 + t * gh * gv * 2, flops)


def bench_latent():
    """Kernels of latent-attention models with experts beside the like kernels
    and products of the uniform families, at 7b sizes."""
    from substratus_amd.models.layers import (LatentAttentionSpec, MoESpec,
                                              RotarySpec)
    from substratus_amd.ops import hybrid as hy
    from substratus_amd.serve.batch import StepBatch
    torch.manual_seed(0)
    bf = dict(device="cuda", dtype=torch.bfloat16)
    F = torch.nn.functional
    h, d, r, rank, w = 32, 128, 64, 512, 4096
    spec = LatentAttentionSpec(h, d, r, d, rank, (d + r) ** -0.5,
                               RotarySpec(1e4, r), None, True)
    moe = MoESpec(32, 8, 2048, 8, 4)

    def batch_of(n, first, tokens):
        need = (first + tokens + 15) // 16
        return StepBatch.build(
            [([1] * tokens, first, list(range(i * need, (i + 1) * need)), i,
              []) for i in range(n)], 16, torch.device("cuda"))

    for rows in (64, 256, 16384):
        it = 100 if rows < 1000 else 20
        x, xf = torch.randn(rows, w, **bf), torch.randn(rows, w,
                                                        device="cuda")
        w32 = torch.randn(w, device="cuda")
        res, wt = torch.randn(rows, w, **bf), torch.randn(w, **bf)
        report(f"rms_norm_residual rows={rows} w={w}",
               timeit(lambda: ops.rms_norm_residual(x, res, wt, 1e-5), it),
               rows * w * 8)
        report(f"  stream_norm rows={rows} w={w}",
               timeit(lambda: hy.stream_norm(x, xf, w32, None, 0.0, 1e-5), it),
               rows * w * 12)
        at = torch.randperm(rows * 8, device="cuda").int().view(rows, 8)
        pk = hy.Picked(torch.randn(rows * 8, w, **bf), at,
                       torch.rand(rows, 8, device="cuda"))
        report(f"  stream_norm of 8 picks rows={rows} w={w}",
               timeit(lambda: hy.stream_norm(pk, xf, w32, None, 0.0, 1e-5),
                      it), rows * w * 26)
        del pk, res
        kc = torch.zeros((rows + 15) // 16, h, 16, d, **bf)
        vc = torch.zeros_like(kc)
        pos = torch.arange(rows, device="cuda", dtype=torch.int32)
        qkv = torch.randn(rows, 3 * h * d, **bf)
        q, k, v = (qkv[:, i * h * d:(i + 1) * h * d].view(rows, h, d)
                   for i in range(3))
        report(f"rope_kv_append rows={rows} {h}x{d}",
               timeit(lambda: ops.rope_kv_append(q, k, v, pos, kc, vc, pos,
                                                 1e4), it),
               rows * h * d * 2 * 7)
        buf = torch.randn(rows, h * (d + r) + h * d + rank + r, **bf)
        cache = torch.zeros((rows + 15) // 16, 1, 16, spec.row, **bf)
        norm, turns = torch.ones(rank, device="cuda"), spec.rot.turns("cuda")
        report(f"  latent_prepare rows={rows}",
               timeit(lambda: hy.latent_prepare(
                   buf, spec, h * (2 * d + r), norm, 1e-5, turns, pos, cache,
                   pos), it), rows * (h * r * 2 + spec.row * 2) * 2)
        router = torch.randn(moe.experts, w, **bf) * 0.02
        ext = hy._ext()
        z = ext.router_scores(x, router)
        report(f"  router_scores rows={rows} {w}->{moe.experts}",
               timeit(lambda: ext.router_scores(x, router), it),
               rows * w * 2 + router.numel() * 2, 2.0 * rows * w * moe.experts)
        ids = torch.empty(rows, moe.top, device="cuda", dtype=torch.int32)
        wts = torch.empty(rows, moe.top, device="cuda")
        report(f"  moe_select rows={rows} {moe.top}/{moe.experts}",
               timeit(lambda: ext.moe_select(ids, wts, z, moe.groups,
                                             moe.keep), it),
               rows * (moe.experts + 2 * moe.top) * 4)
        packed = rows * moe.top
        tile = ext.moe_tile(packed, moe.experts, True, w, moe.ff)
        i32 = dict(device="cuda", dtype=torch.int32)
        at2, src = torch.empty(rows, moe.top, **i32), torch.empty(packed, **i32)
        start = torch.empty(moe.experts + 1, **i32)
        tiles = torch.empty(1 + 2 * ((packed + tile - 1) // tile + moe.experts),
                            **i32)
        report(f"  moe_sort packed={packed}",
               timeit(lambda: ext.moe_sort(at2, src, start, tiles, ids, tile),
                      it), packed * 12)
        up = torch.randn(moe.experts, moe.ff, w, **bf) * 0.02
        down = torch.randn(moe.experts, w, moe.ff, **bf) * 0.02
        hid, out = torch.empty(packed, moe.ff, **bf), torch.empty(packed, w,
                                                                  **bf)
        ff = 11008
        dense = torch.randn(2 * ff, w, **bf) * 0.02
        report(f"linear rows={rows} {w}->{2 * ff}",
               timeit(lambda: F.linear(x, dense), it),
               dense.numel() * 2 + rows * (w + 2 * ff) * 2,
               2.0 * rows * dense.numel())
        dn = torch.randn(w, ff, **bf) * 0.02
        y = torch.randn(rows, ff, **bf)
        report(f"linear rows={rows} {ff}->{w}",
               timeit(lambda: F.linear(y, dn), it),
               dn.numel() * 2 + rows * (w + ff) * 2, 2.0 * rows * dn.numel())
        live = int((start[1:] > start[:-1]).sum())
        wb = live * moe.ff * w * 2
        report(f"  expert_linear up packed={packed} {w}->{moe.ff} "
               f"x{live}", timeit(lambda: ext.expert_linear(
                   hid, x, up, src, start, tiles, tile, "gelu", 0.0), it),
               wb + rows * w * 2 + packed * moe.ff * 2,
               2.0 * packed * w * moe.ff)
        report(f"  expert_linear down packed={packed} {moe.ff}->{w}",
               timeit(lambda: ext.expert_linear(
                   out, hid, down, None, start, tiles, tile, "none", 0.0),
                   it),
               wb + packed * (moe.ff + w) * 2, 2.0 * packed * w * moe.ff)
        del up, down, hid, out, dense, dn, y
        side = 256
        wg = torch.randn(side, w, **bf) * 0.02
        table = torch.randn(1000, side, **bf)
        tok = torch.randint(0, 1000, (rows,), **i32)
        report(f"linear rows={rows} {w}->{side}",
               timeit(lambda: F.linear(x, wg), it),
               wg.numel() * 2 + rows * (w + side) * 2,
               2.0 * rows * wg.numel())
        report(f"  side_gate rows={rows} {w}->{side}",
               timeit(lambda: hy.side_gate(x, wg, tok, table, 0), it),
               wg.numel() * 2 + rows * (w + 2 * side) * 2,
               2.0 * rows * wg.numel())
        if rows < 1000:
            uk_t = torch.randn(h, rank, d, **bf)
            uv = torch.randn(h, d, rank, **bf)
            gate = torch.randn(rows, h * d, **bf)
            q3 = torch.randn(rows, h, d + r, **bf)
            o3 = torch.randn(rows, h, rank, **bf)
            report(f"  head_linear in rows={rows} {h}x{d}->{rank}",
                   timeit(lambda: hy.head_linear(q3, uk_t, tail=r), it),
                   (uk_t.numel() + rows * h * (d + rank + 2 * r)) * 2)
            report(f"  head_linear out rows={rows} {h}x{rank}->{d}",
                   timeit(lambda: hy.head_linear(o3, uv, gate), it),
                   (uv.numel() + rows * h * (2 * d + rank)) * 2)

    for b, ctx in ((8, 512), (64, 512), (256, 512), (16, 3072), (64, 4096)):
        sb = batch_of(b, ctx - 1, 1)
        nb = b * ctx // 16
        cache = torch.randn(nb, 1, 16, spec.row, **bf)
        qa = torch.randn(b, h * spec.row, **bf)
        kc = torch.randn(nb, h, 16, d, **bf)
        vc = torch.randn_like(kc)
        bt = torch.arange(nb, device="cuda", dtype=torch.int32).view(b, -1)
        lens = torch.full((b,), ctx, device="cuda", dtype=torch.int32)
        q = torch.randn(b, h, d, **bf)
        report(f"paged_attn_decode b={b} ctx={ctx} {h}/{h}x{d}",
               timeit(lambda: ops.paged_attn_decode(q, kc, vc, bt, lens,
                                                    d ** -0.5), 50),
               2 * b * ctx * h * d * 2)
        del kc, vc
        o = torch.empty(b, h * rank, **bf)
        report(f"  attn_latent single b={b} ctx={ctx} {h}x{spec.row}",
               timeit(lambda: hy._ext().attn_ctx(
                   o, qa, None, cache, cache[..., :rank], None, None,
                   sb.positions, None, sb.block_table, spec.scale, 0, 0, 0,
                   0.0, 1.0, 1, ctx, False, None, None, None), 50),
               b * ctx * spec.row * 2 + b * h * (spec.row + rank) * 2,
               2.0 * b * ctx * h * (spec.row + rank))

    for b, s_ in ((32, 512), (8, 2048), (4, 4096)):
        t = b * s_
        q, k, v = (torch.randn(t, h, d, **bf) for _ in range(3))
        ss = torch.arange(0, t + 1, s_, dtype=torch.int32, device="cuda")
        report(f"attn_v5 b={b} s={s_} {h}x{d}",
               timeit(lambda: ops.attn_prefill(q, k, v, ss, d ** -0.5), 20),
               4 * t * h * d * 2, 4.0 * b * h * (s_ * (s_ + 1) / 2) * d)
        del q, k, v
        sb = batch_of(b, 0, s_)
        q2 = torch.randn(t, h * (d + r), **bf)
        gate = torch.randn(t, h * d, **bf)
        kv, kr = torch.randn(t, 2 * h * d, **bf), torch.randn(t, r, **bf)
        o = torch.empty(t, h * d, **bf)
        flops = b * h * s_ * (s_ + 1) * (2 * d + r)
        report(f"  attn_flat b={b} s={s_} {h}x{d}+{r}",
               timeit(lambda: hy._ext().attn_flat(
                   o, q2, gate, kv, kr, sb.positions, sb.seq_start,
                   sb.ctx_start, h, d, spec.scale, 0, s_), 20),
               t * (h * (5 * d + r) + r) * 2, flops)
        cache = torch.randn(t // 16, 1, 16, spec.row, **bf)
        c = torch.empty(t, rank, **bf)
        report(f"  latent_gather keys={t}",
               timeit(lambda: hy._ext().latent_gather(
                   c, kr, cache, sb.block_table, sb.ctx_start, sb.positions,
                   sb.seq_start, 0, s_), 20),
               t * spec.row * 4)
        del q2, gate, kv, o, cache
    for b, first, n in ((16, 2048, 16), (4, 4096, 64)):
        sb = batch_of(b, first, n)
        cache = torch.randn(b * (first + n) // 16, 1, 16, spec.row, **bf)
        qa = torch.randn(b * n, h * spec.row, **bf)
        o = torch.empty(b * n, h * rank, **bf)
        report(f"  attn_latent portions b={b} {n} after {first}",
               timeit(lambda: hy._ext().attn_ctx(
                   o, qa, None, cache, cache[..., :rank], None, None,
                   sb.positions, sb.seq_start, sb.block_table, spec.scale, 0,
                   0, 0, 0.0, 1.0, n, first + n, False, None, None, None),
                   20),
               b * (first + n) * spec.row * 2 + b * n * h * 2 * (
                   spec.row + rank),
               2.0 * b * n * (first + n / 2) * h * (spec.row + rank))


EXP = 256 * 16 * 2.4e9    # exponentials/s of the vector units
FMA = 256 * 64 * 2.4e9    # 32-bit vector instructions/s, unpacked


def bench_mixers():
    """Kernels of models with recurrent mixers, windowed attention and gated
    experts beside the like kernels of Kakovik and Guronex, at 7b sizes."""
    from substratus_amd.models.layers import GluSpec, MoESpec, RotarySpec
    from substratus_amd.ops import hybrid as hy
    from substratus_amd.serve.batch import StepBatch
    torch.manual_seed(0)
    bf = dict(device="cuda", dtype=torch.bfloat16)
    f32 = dict(device="cuda")

    def batch_of(n, first, tokens):
        need = (first + tokens + 15) // 16
        return StepBatch.build(
            [([1] * tokens, first, list(range(i * need, (i + 1) * need)), i,
              []) for i in range(n)], 16, torch.device("cuda"))

    w, h, d, inner, ns, rank = 4096, 32, 128, 8192, 16, 256
    for rows in (64, 256, 16384):
        it = 200 if rows < 1000 else 30
        x, xf = torch.randn(rows, w, **bf), torch.randn(rows, w, **f32)
        w32 = torch.randn(w, **f32)
        report(f"stream_norm rows={rows} w={w}",
               timeit(lambda: hy.stream_norm(x, xf, w32, w32, 1.0, 1e-5), it),
               rows * w * 12)
        at = torch.randperm(rows * 8, device="cuda").int().view(rows, 8)
        pk = hy.Picked(torch.randn(rows * 8, w, **bf), at,
                       torch.rand(rows, 8, device="cuda"))
        report(f"stream_norm of 8 picks rows={rows} w={w}",
               timeit(lambda: hy.stream_norm(pk, xf, w32, None, 0.0, 1e-5),
                      it), rows * w * 26)
        report(f"  add_norm rows={rows} w={w}",
               timeit(lambda: hy.add_norm(xf, w32, w32, 1e-5, x.dtype, x), it),
               rows * w * 12)
        report(f"  add_norm and 8 picks rows={rows} w={w}",
               timeit(lambda: hy.add_norm(xf, w32, w32, 1e-5, x.dtype, x, pk),
                      it), rows * w * 28)
        del pk
        buf = torch.randn(rows, 3 * h * d + 32, **bf)
        kc = torch.zeros((rows + 15) // 16, h, 16, d, **bf)
        vc, vf = torch.zeros_like(kc), torch.randn(rows, h * d, **bf)
        pos = torch.arange(rows, device="cuda", dtype=torch.int32)
        wn, lam = torch.ones(h * d, **f32), torch.tensor(0.5, device="cuda")
        report(f"qkv_prepare rows={rows} {h}x{d}",
               timeit(lambda: hy.qkv_prepare(buf, h * d, wn, wn, 1e-5, vf, lam,
                                             kc, vc, pos), it),
               rows * h * d * 2 * 7)
        sb = batch_of(rows, 20, 1) if rows < 1000 else batch_of(8, 0, 2048)
        n = sb.state_slots.numel()
        kc = torch.zeros(rows * 2 if rows < 1000 else rows // 16, h, 16, d,
                         **bf)
        vc = torch.zeros_like(kc)
        cs = torch.zeros(n, 3, 2 * h * d, **bf)
        cw, cb = torch.randn(2 * h * d, 4, **f32), torch.randn(2 * h * d,
                                                               **f32)
        rot = RotarySpec(1e4, d, True)
        turns = rot.turns("cuda")
        rope = hy.rope_table(sb, rot, turns, {})
        taps = n * 3 * 2 * h * d * 4
        report(f"  conv_rope rows={rows} {h}x{d} 4 taps",
               timeit(lambda: hy.conv_rope(buf, cb, cw, cs, rope, kc, vc, sb),
                      it), rows * h * d * 2 * 5 + taps + rows * d * 4)
        for ch in (3 * h * d, inner):
            cs = torch.zeros(n, 3, ch, **bf)
            cw, x2 = torch.randn(ch, 4, **f32), torch.randn(rows, ch, **bf)
            report(f"  short_conv rows={rows} {ch} 4 taps",
                   timeit(lambda: hy.short_conv(x2, cw, None, True, cs, sb),
                          it), rows * ch * 4 + n * 3 * ch * 4)
        up = torch.randn(rows, 2 * 11008, **bf)
        report(f"silu_mul rows={rows} 11008",
               timeit(lambda: hy.silu_mul(up), it), rows * 11008 * 6)
        out = torch.empty(rows, 11008, **bf)
        report(f"  glu relu rows={rows} 11008",
               timeit(lambda: hy.glu(up, GluSpec("relu"), out), it),
               rows * 11008 * 6)
        o, nw = torch.randn(rows, h * d, **bf), torch.ones(h * d, **f32)
        report(f"  joint_gate rows={rows} {h * d}",
               timeit(lambda: hy.joint_gate(o, nw, up[:, :h * d], 1e-5, x),
                      it), rows * h * d * 6)
        for k, n2 in ((rank, inner), (d, h * d)):
            low, wl = torch.randn(rows, k, **bf), torch.randn(n2, k, **bf)
            report(f"  linear32 rows={rows} {k}->{n2}",
                   timeit(lambda: hy.linear32(low, wl), it),
                   (rows * k + n2 * k) * 2 + rows * n2 * 4,
                   2.0 * rows * k * n2)
        for name, moe, f in (
                ("gelu 8 of 32 x 2048", MoESpec(32, 8, 2048, 8, 4), 1),
                ("gated 8 of 32 x 1024", MoESpec(
                    32, 8, 1024, glu=GluSpec("clamped", 7.0),
                    over_chosen=True), 2)):
            wu = torch.randn(32, f * moe.ff, w, **bf) * 0.02
            wd = torch.randn(32, w, moe.ff, **bf) * 0.02
            router = torch.randn(32, w, **bf) * 0.02
            report(f"{'  ' if f == 2 else ''}experts rows={rows} {name}",
                   timeit(lambda: hy.experts(x, router, wu, wd, moe), it),
                   (wu.numel() + wd.numel() + rows * 8 * (w + 2 * moe.ff)) * 2,
                   2.0 * rows * 8 * moe.ff * w * (f + 1))
            del wu, wd
        del buf, kc, vc, up

    sink = torch.zeros(h, **f32)
    bias = torch.randn(h, 4096, **f32)
    for b, ctx in ((8, 512), (64, 512), (256, 512), (64, 2048)):
        nb = b * ctx // 16
        kc = torch.randn(nb, h, 16, d, **bf)
        vc, q = torch.randn_like(kc), torch.randn(b, h * d, **bf)
        sb, gate = batch_of(b, ctx - 1, 1), torch.randn(b, h, **bf)
        report(f"attn_ctx single b={b} ctx={ctx} chunk",
               timeit(lambda: hy.attn_ctx(q, gate, kc, vc, bias, sb,
                                          d ** -0.5, 4096), 100),
               4 * b * ctx * h * d)
        report(f"  attn_ctx single b={b} ctx={ctx} window 1024, cap, sink",
               timeit(lambda: hy.attn_ctx(
                   q, None, kc, vc, None, sb, d ** -0.5, window=1024, keep=4,
                   softcap=30.0, sink=sink), 100),
               4 * b * min(ctx, 1028) * h * d)
        del kc, vc
    for b, s_ in ((32, 512), (8, 2048), (4, 4096)):
        t = b * s_
        q, kc = torch.randn(t, h * d, **bf), torch.randn(t // 16, h, 16, d,
                                                         **bf)
        vc, sb = torch.randn_like(kc), batch_of(b, 0, s_)
        gate, k = torch.randn(t, h, **bf), min(s_, 1024)
        report(f"attn_ctx portions b={b} s={s_} chunk",
               timeit(lambda: hy.attn_ctx(q, gate, kc, vc, bias, sb,
                                          d ** -0.5, 4096), 20),
               8 * t * h * d, 4.0 * b * h * (s_ * (s_ + 1) / 2) * d)
        report(f"  attn_ctx portions b={b} s={s_} window 1024, cap, sink",
               timeit(lambda: hy.attn_ctx(
                   q, None, kc, vc, None, sb, d ** -0.5, window=1024, keep=4,
                   softcap=30.0, sink=sink), 20), 8 * t * h * d,
               4.0 * b * h * d * (k * (k + 1) / 2 + (s_ - k) * (k + 4)))
        del q, kc, vc

    gh, gv = 16, 256
    a2, ab = torch.randn(gh * d, 16, **f32) * 0.25, torch.randn(gh * d, **f32)
    nw, nv = torch.ones(gv, **f32), torch.ones(d, **f32)
    decay = torch.full((h,), 0.99, **f32)
    rate, zb = torch.full((h,), 0.5, **f32), torch.full((h * d,), -4.0, **f32)
    la, ld_ = -torch.rand(inner, ns, **f32) * 8, torch.ones(inner, **f32)
    zs = torch.full((inner,), -4.0, **f32)
    for b, s_ in ((8, 1), (64, 1), (256, 1), (32, 512), (8, 2048), (1, 8192)):
        t, it = b * s_, 100 if s_ == 1 else 20
        sb = batch_of(b, 100 if s_ == 1 else 0, s_)
        what = f"single b={b}" if s_ == 1 else f"portions b={b} s={s_}"
        c = 32.0 if s_ > 1 else 0.0
        # state products and, within chunks of 32, score products
        state, x = torch.zeros(b, gh, d, gv, **f32), torch.randn(
            t, 2 * gh * (d + gv) + 16, **bf)
        held = state.numel() * 8
        report(f"gla {what} {gh}x{d}x{gv}",
               timeit(lambda: hy.gla(x, a2, ab, nw, state, sb, 16.0, 1e-5),
                      it), held + x.numel() * 2 + t * gh * gv * 2,
               t * gh * (4.0 * d * gv + c * (d + gv)) if s_ > 1 else 0)
        state, x = torch.zeros(b, h, d, d, **f32), torch.randn(
            t, 4 * h * d, **bf)
        report(f"  lightning {what} {h}x{d}x{d}",
               timeit(lambda: hy.lightning(x, decay, state, sb), it),
               held + t * h * d * 8,
               t * h * (4.0 * d * d + c * 2 * d) if s_ > 1 else 0)
        x = torch.randn(t, 3 * h * d, **bf)
        z, beta = torch.randn(t, h * d, **f32), torch.randn(t, h, **bf)
        gate, out = torch.randn(t, h * d, **bf), torch.empty(t, h * d, **bf)
        report(f"  delta {what} {h}x{d}x{d}",
               timeit(lambda: hy.delta(x, z, zb, rate, beta, nv, gate, state,
                                       sb, h, 1e-5, 1.0, out), it),
               held + t * h * d * 14,
               t * h * (6.0 * d * d + c * 4 * d) if s_ > 1 else 0)
        state = torch.zeros(b, inner, ns, **f32)
        u, g = torch.randn(t, inner, **bf), torch.randn(t, 2 * inner, **bf)
        z, o = torch.randn(t, inner, **f32), torch.empty(t, inner, **bf)
        low = torch.randn(t, rank + 2 * ns, **bf)
        # one exponential and four other instructions per state and token
        steps = t * inner * ns
        report(f"  selective_scan {what} {inner}x{ns}",
               timeit(lambda: hy.selective_scan(
                   u, g[:, inner:], z, zs, low, rank, la, ld_, state, sb, o),
                   it),
               max(state.numel() * 8 + t * inner * 10,
                   HBM * steps * (1 / EXP + 4 / FMA)))


def bench_sigmoid():
    """Kernels of sigmoid attention behind convolutions, of windowed latent
    attention and of corrected routers beside the like kernels of Kakovik,
    Guronex and Vurazen, at 7b sizes."""
    from substratus_amd.models.layers import (GluSpec, LatentAttentionSpec,
                                              MoESpec, QueryTemperature,
                                              RotarySpec)
    from substratus_amd.ops import hybrid as hy
    from substratus_amd.serve.batch import StepBatch
    torch.manual_seed(0)
    bf = dict(device="cuda", dtype=torch.bfloat16)
    f32, i32 = dict(device="cuda"), dict(device="cuda", dtype=torch.int32)
    ext = hy._ext()

    def batch_of(n, first, tokens):
        need = (first + tokens + 15) // 16
        return StepBatch.build(
            [([1] * tokens, first, list(range(i * need, (i + 1) * need)), i,
              []) for i in range(n)], 16, torch.device("cuda"))

    w, h, d, r, rank, q_rank, win = 4096, 32, 128, 64, 512, 1536, 1024
    old = LatentAttentionSpec(h, d, r, d, rank, (d + r) ** -0.5,
                              RotarySpec(1e4, r), None, True)
    new = LatentAttentionSpec(h, d, 0, d, rank, d ** -0.5, None,
                              head_gate=True, q_rank=q_rank, window=win)
    temp = QueryTemperature(0.1, 1024)
    for rows in (64, 256, 16384):
        it = 200 if rows < 1000 else 30
        sb = batch_of(rows, 20, 1) if rows < 1000 else batch_of(8, 0, 2048)
        n = sb.state_slots.numel()
        table, vecs = torch.randn(32000, w, **bf), torch.randn(8192, w, **bf)
        w32 = torch.randn(w, **f32)
        tok = torch.randint(0, 32000, (rows,), **i32)
        report(f"embed_norm rows={rows} w={w}",
               timeit(lambda: hy.embed_norm(tok, table, w32, 1.0, 1e-5), it),
               rows * w * 8)
        report(f"  embed_norm with positions rows={rows} w={w}",
               timeit(lambda: hy.embed_norm(tok, table, w32, 1.0, 1e-5, 64.0,
                                            vecs, sb.positions), it),
               rows * w * 10)
        del table, vecs
        x = torch.randn(rows, w, **bf)
        pages = rows * 2 if rows < 1000 else rows // 16
        kc = torch.zeros(pages, h, 16, d, **bf)
        vc = torch.zeros_like(kc)
        buf = torch.randn(rows, 3 * h * d, **bf)
        for name, parts in (("conv_rope", 2), ("  conv_qkv", 3)):
            ch = parts * h * d
            cs = torch.zeros(n, 3, ch, **bf)
            cw, cb = torch.randn(ch, 4, **f32), torch.randn(ch, **f32)
            taps = n * 3 * ch * 4
            if parts == 2:
                rot = RotarySpec(1e4, d, True)
                rope = hy.rope_table(sb, rot, rot.turns("cuda"), {})
                dt = timeit(lambda: hy.conv_rope(buf, cb, cw, cs, rope, kc, vc,
                                                 sb), it)
                nbytes = rows * h * d * 2 * 5 + taps + rows * d * 4
            else:
                dt = timeit(lambda: hy.conv_qkv(buf, cb, cw, cs, kc, vc, sb,
                                                temp, 1e-5), it)
                nbytes = rows * h * d * 2 * 6 + taps
            report(f"{name} rows={rows} {h}x{d} 4 taps", dt, nbytes)
        del kc, vc, buf
        pos = torch.arange(rows, **i32)
        norm, qn = torch.ones(rank, **f32), torch.ones(q_rank, **f32)
        buf = torch.randn(rows, h * (2 * d + r) + rank + r, **bf)
        cache = torch.zeros((rows + 15) // 16, 1, 16, old.row, **bf)
        turns = old.rot.turns("cuda")
        report(f"latent_prepare rows={rows}",
               timeit(lambda: hy.latent_prepare(
                   buf, old, h * (2 * d + r), norm, 1e-5, turns, pos, cache,
                   pos), it), rows * (h * r * 2 + old.row * 2) * 2)
        buf = torch.randn(rows, q_rank + rank + h, **bf)
        cache = torch.zeros((rows + 15) // 16, 1, 16, rank, **bf)
        turns = torch.empty(0, dtype=torch.float64, device="cuda")
        report(f"  latent_prepare with queries' latent rows={rows}",
               timeit(lambda: hy.latent_prepare(
                   buf, new, q_rank, norm, 1e-5, turns, pos, cache, pos, qn),
                   it), rows * (q_rank + rank) * 4)
        corr = torch.randn(32, **f32) * 0.01
        gates = torch.randn(rows, h * d, **bf)
        if rows < 1000:
            uv = torch.randn(h, d, rank, **bf)
            o3 = torch.randn(rows, h, rank, **bf)
            for name, g in (("head_linear out", gates),
                            ("  head_linear out, gate per head",
                             gates[:, :h])):
                report(f"{name} rows={rows} {h}x{rank}->{d}",
                       timeit(lambda: hy.head_linear(o3, uv, g), it),
                       (uv.numel() + rows * h * (d + rank) + g.numel()) * 2)
        for name, moe, f in (
                ("8 of 32 x 1024", MoESpec(
                    32, 8, 1024, 8, 4, glu=GluSpec("clamped", 7.0)), 0),
                ("8 of 32 x 1344", MoESpec(
                    32, 8, 1344, 8, 4, GluSpec("silu"), sigmoid=True,
                    correction=True, group_best=2), 1)):
            z = torch.randn(1, rows, 32, **f32)
            ids = torch.empty(rows, 8, **i32)
            wts = torch.empty(rows, 8, **f32)
            report(f"{'  ' * f}moe_select{' corrected' * f} rows={rows} 8/32",
                   timeit(lambda: ext.moe_select(
                       ids, wts, z, 8, 4, None, False, moe.sigmoid,
                       corr if f else None, moe.group_best), it),
                   rows * (32 + 16) * 4)
            wu = torch.randn(32, 2 * moe.ff, w, **bf) * 0.02
            wd = torch.randn(32, w, moe.ff, **bf) * 0.02
            router = torch.randn(32, w, **bf) * 0.02
            report(f"{'  ' * f}experts rows={rows} {name}",
                   timeit(lambda: hy.experts(x, router, wu, wd, moe, None,
                                             corr if f else None), it),
                   (wu.numel() + wd.numel() + rows * 8 * (w + 2 * moe.ff)) * 2,
                   6.0 * rows * 8 * moe.ff * w)
            del wu, wd

    fall = torch.full((h,), 0.5, **f32), torch.full((h,), 0.5, **f32)
    wb, bias = torch.full((h,), -4.0, **f32), torch.randn(h, 4096, **f32)
    for b, ctx, kv in ((8, 512, h), (64, 512, h), (256, 512, h),
                       (64, 2048, h), (64, 2048, 8), (64, 2048, 1)):
        nb = b * ctx // 16
        kc = torch.randn(nb, kv, 16, d, **bf)
        vc, q = torch.randn_like(kc), torch.randn(b, h * d, **bf)
        sb, gate = batch_of(b, ctx - 1, 1), torch.randn(b, h, **bf)
        what = f"single b={b} ctx={ctx} {h}/{kv}x{d}"
        report(f"attn_ctx {what} softmax, chunk, bias",
               timeit(lambda: hy.attn_ctx(q, gate, kc, vc, bias, sb,
                                          d ** -0.5, 4096), 100),
               4 * b * ctx * kv * d, 4.0 * b * ctx * h * d)
        report(f"  attn_ctx {what} sigmoid, falloff",
               timeit(lambda: hy.attn_ctx(
                   q, None, kc, vc, None, sb, d ** -0.5, falloff=fall,
                   weight_bias=wb), 100),
               4 * b * ctx * kv * d, 4.0 * b * ctx * h * d)
        del kc, vc
    for b, ctx in ((8, 512), (64, 512), (256, 512), (16, 3072), (64, 4096)):
        sb = batch_of(b, ctx - 1, 1)
        for name, spec in (("", old), ("  ", new)):
            row, seen = spec.row, min(spec.window or ctx, ctx)
            cache = torch.randn(b * ctx // 16, 1, 16, row, **bf)
            qa, o = torch.randn(b, h * row, **bf), torch.empty(b, h * rank,
                                                               **bf)
            report(f"{name}attn_latent single b={b} ctx={ctx} {h}x{row}"
                   f"{' window 1024' if spec.window else ''}",
                   timeit(lambda: ext.attn_ctx(
                       o, qa, None, cache, cache[..., :rank], None, None,
                       sb.positions, None, sb.block_table, spec.scale, 0,
                       spec.window, 0, 0.0, 1.0, 1, seen, False, None, None,
                       None), 50),
                   b * seen * row * 2 + b * h * (row + rank) * 2,
                   2.0 * b * seen * h * (row + rank))
            del cache
    for b, s_ in ((32, 512), (8, 2048), (4, 4096)):
        t = b * s_
        q, kc = torch.randn(t, h * d, **bf), torch.randn(t // 16, h, 16, d,
                                                         **bf)
        vc, sb = torch.randn_like(kc), batch_of(b, 0, s_)
        gate = torch.randn(t, h, **bf)
        flops = 4.0 * b * h * (s_ * (s_ + 1) / 2) * d
        report(f"attn_ctx portions b={b} s={s_} softmax, chunk, bias",
               timeit(lambda: hy.attn_ctx(q, gate, kc, vc, bias, sb,
                                          d ** -0.5, 4096), 20),
               8 * t * h * d, flops)
        report(f"  attn_ctx portions b={b} s={s_} sigmoid, falloff",
               timeit(lambda: hy.attn_ctx(
                   q, None, kc, vc, None, sb, d ** -0.5, falloff=fall,
                   weight_bias=wb), 20), 8 * t * h * d, flops)
        del q, kc, vc
        k = min(s_, win)
        for name, spec in (("", old), ("  ", new)):
            dq, r_ = d + spec.rot_dim, spec.rot_dim
            q = torch.randn(t, h * dq, **bf)
            kv, kr = torch.randn(t, 2 * h * d, **bf), torch.randn(t, r_, **bf)
            o = torch.empty(t, h * d, **bf)
            g = torch.randn(t, h * d if spec.out_gate else h, **bf)
            pairs = k * (k + 1) / 2 + (s_ - k) * k if spec.window else \
                s_ * (s_ + 1) / 2
            report(f"{name}attn_flat b={b} s={s_} {h}x{d}+{r_}"
                   f"{' window 1024' if spec.window else ''}",
                   timeit(lambda: ext.attn_flat(
                       o, q, g, kv, kr, sb.positions, sb.seq_start,
                       sb.context(spec.window)[0], h, d, spec.scale,
                       spec.window, s_), 20),
                   (t * (h * (4 * d + r_) + r_) + g.numel()) * 2,
                   2.0 * b * h * pairs * (2 * d + r_))
            cache = torch.randn(t // 16, 1, 16, spec.row, **bf)
            c = torch.empty(t, rank, **bf)
            report(f"{name}latent_gather keys={t} of {spec.row}",
                   timeit(lambda: ext.latent_gather(
                       c, kr, cache, sb.block_table,
                       sb.context(spec.window)[0], sb.positions, sb.seq_start,
                       spec.window, s_), 20), t * spec.row * 4)
            del q, kv, o, cache


def bench_sample(B=64, V=32000):
    logits = torch.randn(B, V, device="cuda").bfloat16()
    temp = torch.zeros(B, device="cuda")
    tk = torch.zeros(B, dtype=torch.int32, device="cuda")
    tp = torch.ones(B, device="cuda")
    u = torch.rand(B, device="cuda")
    dt = timeit(lambda: ops.softmax_sample(logits, temp, tk, tp, u))
    print(f"softmax_sample greedy B={B} V={V}: {dt*1e6:.1f} us")


def bench_prefill(B=8, hq=32, hkv=32, d=128, S=512):
    torch.manual_seed(0)
    t = B * S
    q = torch.randn(t, hq, d, device="cuda").bfloat16()
    k = torch.randn(t, hkv, d, device="cuda").bfloat16()
    v = torch.randn(t, hkv, d, device="cuda").bfloat16()
    ss = torch.arange(0, t + 1, S, dtype=torch.int32, device="cuda")
    scale = d ** -0.5
    dt = timeit(lambda: ops.attn_prefill(q, k, v, ss, scale), iters=50)
    flops = 4.0 * B * hq * (S * (S + 1) / 2) * d
    print(f"attn_prefill B={B} S={S} hq={hq} d={d}: {dt*1e6:.1f} us, "
          f"{flops/dt/1e12:.0f} TF/s")


def bench_prefill_ablation(B=8, S=512, hq=32, hkv=32, d=128):
    """Within-probe variant ablation (guide rule 8): where does prefill time
    go? Variants are timing-only (wrong numerics)."""
    from substratus_amd import _C
    torch.manual_seed(0)
    t = B * S
    q = torch.randn(t, hq, d, device="cuda").bfloat16()
    k = torch.randn(t, hkv, d, device="cuda").bfloat16()
    v = torch.randn(t, hkv, d, device="cuda").bfloat16()
    out = torch.empty_like(q)
    ss = torch.arange(0, t + 1, S, dtype=torch.int32, device="cuda")
    names = {0: "full", 1: "no-softmax-valu", 2: "no-pv-mfma",
             3: "no-v-staging", 4: "no-qk-mfma"}
    flops = 4.0 * B * hq * (S * (S + 1) / 2) * d
    for variant in (0, 1, 2, 3, 4):
        dt = timeit(lambda: _C.attn_prefill_probe(variant, out, q, k, v, ss,
                                                  S, d ** -0.5), iters=50)
        print(f"prefill variant {variant} ({names[variant]:16s}): "
              f"{dt*1e6:7.1f} us  ({flops/dt/1e12:4.0f} TF-equiv)")


def bench_decode_gemm(m=256):
    import torch.nn.functional as F
    from substratus_amd import _C
    shapes = [(12288, 4096), (4096, 4096), (22016, 4096), (4096, 11008)]
    for n, k in shapes:
        torch.manual_seed(0)
        x = torch.randn(m, k, device="cuda").bfloat16()
        w = torch.randn(n, k, device="cuda").bfloat16() * 0.02
        y = torch.empty(m, n, device="cuda").bfloat16()
        dt_ours = timeit(lambda: _C.decode_gemm(y, x, w), iters=100)
        dt_blas = timeit(lambda: F.linear(x, w), iters=100)
        wb = n * k * 2
        print(f"decode_gemm M={m} N={n} K={k}: ours {dt_ours*1e6:.1f} us "
              f"({wb/dt_ours/1e12:.2f} TB/s W) vs hipBLASLt "
              f"{dt_blas*1e6:.1f} us ({wb/dt_blas/1e12:.2f} TB/s)")


def bench_wstream(m=256):
    """wstream GEMM v2 vs hipBLASLt, interleaved rounds (guide rule 24),
    plus a parity check against fp32 matmul. Shapes: llama2-7b decode
    projections + the logits GEMM."""
    import torch.nn.functional as F
    from substratus_amd import ops
    from substratus_amd import _C
    shapes = [(12288, 4096), (4096, 4096), (22016, 4096), (4096, 11008),
              (32000, 4096)]
    for n, k in shapes:
        torch.manual_seed(0)
        x = (torch.randn(m, k, device="cuda") * 0.3).bfloat16()
        w = (torch.randn(n, k, device="cuda") * 0.02).bfloat16()
        wp = ops.wstream_repack(w)
        y = ops.wstream_linear(x, wp, n, k)
        refy = (x.float() @ w.float().T)
        err = (y.float() - refy).abs().max().item()
        scale = refy.abs().max().item()
        ok = err <= 0.02 * max(scale, 1.0)
        # interleaved timing rounds
        ours, blas = [], []
        for _ in range(5):
            ours.append(timeit(lambda: ops.wstream_linear(x, wp, n, k),
                               iters=50))
            blas.append(timeit(lambda: F.linear(x, w), iters=50))
        do, db = min(ours), min(blas)
        wb = n * k * 2
        print(f"wstream M={m} N={n} K={k}: ours {do*1e6:6.1f} us "
              f"({wb/do/1e12:.2f} TB/s W) vs hipBLASLt {db*1e6:6.1f} us "
              f"({wb/db/1e12:.2f} TB/s)  x{db/do:.2f}  "
              f"parity={'OK' if ok else f'FAIL err={err:.4f}/{scale:.1f}'}")


def bench_attn_v5():
    """V4 vs V5 prefill attention, interleaved rounds (guide rule 24), on
    the serving (llama2-7b) and training (falcon) shapes."""
    from substratus_amd import _C
    shapes = [("llama S512", 8, 32, 32, 128, 512),
              ("llama S2048", 4, 32, 32, 128, 2048),
              ("falcon S2048", 4, 71, 1, 64, 2048)]
    for name, B, hq, hkv, d, S in shapes:
        torch.manual_seed(0)
        t = B * S
        q = (torch.rand(t, hq, d, device="cuda") * 2 - 1).bfloat16()
        k = (torch.rand(t, hkv, d, device="cuda") * 2 - 1).bfloat16()
        v = (torch.rand(t, hkv, d, device="cuda") * 2 - 1).bfloat16()
        ss = torch.arange(0, (B + 1) * S, S, dtype=torch.int32,
                          device="cuda")
        out = torch.empty_like(q)
        scale = d ** -0.5
        t4, t5 = [], []
        for _ in range(5):
            t4.append(timeit(lambda: _C.attn_prefill(
                out, q, k, v, ss, S, scale), iters=30))
            t5.append(timeit(lambda: _C.attn_v5(
                out, q, k, v, ss, S, scale, None), iters=30))
        flops = 2 * 2 * B * hq * S * S * d * 0.5
        print(f"attn {name}: v4 {min(t4)*1e6:.0f} us "
              f"({flops/min(t4)/1e12:.0f} TF) vs v5 {min(t5)*1e6:.0f} us "
              f"({flops/min(t5)/1e12:.0f} TF)")


def bench_attn_bwd():
    """Backward kernels old-vs-V5, interleaved (falcon MQA + llama
    shapes) — the dkv_v5 slowdown diagnosis harness."""
    from substratus_amd import _C
    shapes = [("falcon", 4, 71, 1, 64, 2048), ("llama", 4, 32, 32, 128, 2048)]
    for name, B, hq, hkv, d, S in shapes:
        torch.manual_seed(0)
        t = B * S
        q = (torch.rand(t, hq, d, device="cuda") * 2 - 1).bfloat16()
        k = (torch.rand(t, hkv, d, device="cuda") * 2 - 1).bfloat16()
        v = (torch.rand(t, hkv, d, device="cuda") * 2 - 1).bfloat16()
        do = torch.randn_like(q)
        ss = torch.arange(0, (B + 1) * S, S, dtype=torch.int32,
                          device="cuda")
        out = torch.empty_like(q)
        lse = torch.empty(t, hq, dtype=torch.float32, device="cuda")
        scale = d ** -0.5
        _C.attn_v5(out, q, k, v, ss, S, scale, lse)
        dq = torch.empty_like(q)
        dk = torch.zeros(t, hkv, d, dtype=torch.float32, device="cuda")
        dv = torch.zeros_like(dk)
        delta = torch.empty_like(lse)
        import os as _os
        for tag, env in (("mixed", None), ("dkv_v5", "1")):
            if env: _os.environ["SUB_ATTN_DKV_V5"] = env
            else: _os.environ.pop("SUB_ATTN_DKV_V5", None)
            dt = timeit(lambda: _C.attn_train_bwd_v5(
                dq, dk, dv, q, k, v, out, do, lse, delta, ss, S, scale),
                iters=20)
            print(f"bwd {name} [{tag}]: {dt*1e6:.0f} us")


def bench_mgemm(m=512):
    """mfma_gemm v3 (256x256 glds tile) vs hipBLASLt, interleaved rounds
    (guide rule 24) + parity vs fp32 matmul. Shapes: llama2-7b B=512 decode
    projections + logits."""
    import torch.nn.functional as F
    from substratus_amd import _C, ops
    shapes = [("qkv", 12288, 4096), ("o", 4096, 4096),
              ("gateup", 22016, 4096), ("down", 4096, 11008),
              ("logits", 32000, 4096)]
    for name, n, k in shapes:
        torch.manual_seed(0)
        x = (torch.rand(m, k, device="cuda") * 2 - 1).bfloat16()
        w = ((torch.rand(n, k, device="cuda") * 2 - 1) * 0.02).bfloat16()
        y = torch.empty(m, n, device="cuda").bfloat16()
        splitk = int(_C.mfma_gemm_pick_splitk(m, n, k))
        part = (torch.empty(splitk * m * n, dtype=torch.float32,
                            device="cuda") if splitk > 1 else None)
        _C.mfma_gemm(y, x, w, None, part, splitk)
        ref = (x.float() @ w.float().t())
        err = (y.float() - ref).abs().max().item()
        rel = err / ref.abs().max().item()
        # interleaved A/B rounds
        ours, blas = [], []
        for _ in range(5):
            ours.append(timeit(
                lambda: _C.mfma_gemm(y, x, w, None, part, splitk), iters=50))
            blas.append(timeit(lambda: F.linear(x, w), iters=50))
        dt_o, dt_b = min(ours), min(blas)
        wb = n * k * 2
        print(f"mgemm {name} M={m} N={n} K={k} splitk={splitk}: "
              f"ours {dt_o*1e6:.1f} us ({wb/dt_o/1e12:.2f} TB/s W, "
              f"{2*m*n*k/dt_o/1e12:.0f} TF) vs hipBLASLt {dt_b*1e6:.1f} us "
              f"({wb/dt_b/1e12:.2f} TB/s) | maxerr {err:.4f} rel {rel:.2e}")


def bench_quant_gemv(n=13824, k=5120, quant="q4_0"):
    from substratus_amd.parallel.tp import Linear
    from substratus_amd.models.quant import QuantLinear
    torch.manual_seed(0)
    lin = Linear(k, n, bias=False, dtype=torch.float32)
    lin.weight.data.normal_(0, 0.1)
    ql = QuantLinear.from_linear(lin, quant).to("cuda")
    for m in (1, 4):
        x = torch.randn(m, k, device="cuda").bfloat16()
        dt = timeit(lambda: ql(x))
        wb = ql.qs.numel() + ql.scales.numel() * 2
        print(f"quant_gemv {quant} N={n} K={k} M={m}: {dt*1e6:.1f} us, "
              f"{wb/dt/1e12:.2f} TB/s (weights)")


if __name__ == "__main__":
    ap = argparse.ArgumentParser()
    ap.add_argument("--which", default="all")
    a = ap.parse_args()
    if a.which in ("all", "attn"):
        bench_attn()
        bench_attn(ctx=2048)
        bench_attn(hq=64, hkv=8, ctx=512)  # llama2-70b-style GQA
    if a.which == "attngqa":           # GQA decode sweep (LDS-staged path)
        bench_attn(B=512, hq=32, hkv=32, ctx=512)   # MHA reference point
        bench_attn(B=512, hq=64, hkv=8, ctx=512)    # llama2-70b
        bench_attn(B=256, hq=64, hkv=8, ctx=512)
        bench_attn(B=256, hq=64, hkv=8, ctx=128)    # short-ctx regime
        bench_attn(B=512, hq=64, hkv=8, ctx=2048)
        bench_attn(B=512, hq=128, hkv=8, d=64, ctx=512)  # GQA-16 d=64
        bench_attn(B=64, hq=64, hkv=8, ctx=512)     # nsplit>1 regime
    if a.which in ("all", "prefill"):
        bench_prefill()
        bench_prefill(S=2048, B=4)
    if a.which == "prefill_ablate":
        bench_prefill_ablation()
    if a.which in ("all", "rope"):
        bench_rope()
    if a.which == "hybrid":
        bench_hybrid()
    if a.which == "latent":
        bench_latent()
    if a.which == "mixers":
        bench_mixers()
    if a.which == "sigmoid":
        bench_sigmoid()
    if a.which in ("all", "norm"):
        bench_norm()
    if a.which in ("all", "sample"):
        bench_sample()
    if a.which in ("all", "dgemm"):
        bench_decode_gemm()
        bench_decode_gemm(m=64)
    if a.which in ("all", "wstream"):
        bench_wstream()
        bench_wstream(m=64)
    if a.which in ("all", "attnv5"):
        bench_attn_v5()
    if a.which == "attnbwd":
        bench_attn_bwd()
    if a.which in ("all", "mgemm"):
        m = int(os.environ.get("MGEMM_M", "512"))
        bench_mgemm(m)
    if a.which in ("all", "quant"):
        bench_quant_gemv()
        bench_quant_gemv(quant="q8_0")
