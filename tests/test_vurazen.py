"""Vurazen models through the engine against the plain float64 implementation
in tests/oracles, on the CPU ops and on the GPU kernels."""

import json
import math
import os
import subprocess

import pytest
import torch

from oracles import vurazen as oracle
from oracles import vurazen_models as models
from oracles.harness import (LIMIT, PLACES, TRACE, Replayed, engine_for,
                             error, generate, greedy_share, put, replay_cut,
                             request_batch, tol, written_models)
from substratus_amd.models import get_config
from substratus_amd.models.layers import (GluSpec, LoopSpec, MoESpec,
                                          RotarySpec)
from substratus_amd.models.weights import load_weights
from substratus_amd.ops import hybrid as ops
from substratus_amd.serve.batch import StepBatch
from substratus_amd.serve.engine import Engine, EngineConfig
from substratus_amd.serve.kv_cache import PagedKVCache
from substratus_amd.serve.trace import TraceReplay

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
EVERY_PLACE = pytest.mark.parametrize("place", PLACES)
CUTS = pytest.mark.parametrize("cuts", [
    [70], [1] * 70, [2] * 35, [1, 2, 31, 1, 33, 2], [33, 17, 3, 16, 1]],
    ids=["whole", "singly", "twos", "uneven", "portions"])


@pytest.fixture(scope="module")
def folder(tmp_path_factory):
    """name -> (folder, config, weights)"""
    return written_models(tmp_path_factory, models)


_expected = {}


def expected(cfg, w, toks, key):
    if key not in _expected:
        _expected[key] = oracle.forward(cfg, w, toks)
    return _expected[key]


def check_greedy(cfg, w, prompt, got, dtype):
    return greedy_share(oracle.forward(cfg, w, prompt + got), prompt, got,
                        dtype)


# ---- configuration and registry ---------------------------------------------

def test_config_is_read_from_the_folder(folder):
    cfg = get_config(folder("mixed")[0])
    assert cfg.family == "vurazen" and cfg.num_layers == 5
    assert (cfg.hidden_size, cfg.vocab_size) == (80, 101)
    assert (cfg.embed_scale, cfg.logit_softcap) == (1.5, 9.0)
    assert cfg.loop == LoopSpec(1, 4, 2)
    assert [(i, t) for i, t in cfg.runs()] == \
        oracle.passes(models.CONFIGS["mixed"][0])
    both = cfg.layers[1].mixer
    a, d = both.left, both.right
    assert (both.left_scale, both.right_scale) == (0.7, 1.2)
    assert (a.heads, a.kv_heads, a.dim, a.taps, a.window, a.keep) == \
        (4, 2, 24, 3, 24, 3)
    assert (a.softcap, a.sink, a.rot) == (8.0, True,
                                          RotarySpec(100.0, 12, True))
    assert (d.heads, d.kv_heads, d.dim, d.vdim, d.taps, d.decay_rank,
            d.gate_rank) == (4, 2, 16, 24, 4, 8, 12)
    assert cfg.layers[0].mixer.decay == (0.5, 0.9, 0.995)
    assert cfg.layers[1].glu == GluSpec("relu") and cfg.layers[1].ff == 72
    assert cfg.layers[2].ff == 0 and cfg.layers[2].moe is None
    assert cfg.layers[3].moe == MoESpec(
        6, 3, 32, glu=GluSpec("clamped", 0.8), over_chosen=True, bias=True)
    assert cfg.layers[4].moe.shared_glu == GluSpec("clamped", 0.7)
    assert cfg.layers[4].moe.shared_ff == 24


def test_param_count_matches_the_weights(folder):
    for name in models.CONFIGS:
        d, _, w = folder(name)
        big = sum(t.numel() for n, t in w.items() if t.dim() == 2
                  and n != "loop.step")
        assert get_config(d).param_count() == big


def test_registered_sizes():
    for name in ("vurazen-tiny", "vurazen-1b", "vurazen-7b"):
        cfg = get_config(name)
        assert cfg.layers and cfg.param_count() > 0


@pytest.mark.parametrize("layer", [
    dict(models.mamba(8, 4, 2, 2), type="other"),
    dict(models.mamba(8, 4, 2, 2), mlp={"kind": "other"}),
    models.lightning(2, 8, 8, [0.5]),
    models.both(models.att(3, 2, 8, 2, 9, 0, 4), models.delta(1, 1, 8, 8, 2),
                1, 1),
    models.both(models.att(2, 2, 8, 2, 9, 0, 10), models.delta(1, 1, 8, 8, 2),
                1, 1),
    models.both(models.att(2, 2, 8, 2, 9, 0, 4), models.delta(3, 2, 8, 8, 2),
                1, 1),
    models.both(dict(models.att(2, 2, 8, 2, 9, 0, 4), vdim=6),
                models.delta(1, 1, 8, 8, 2), 1, 1),
    models.moe(models.mamba(8, 4, 2, 2), 3, 4, 8, 1.0)])
def test_what_cannot_be_is_refused(tmp_path, layer):
    (tmp_path / "config.json").write_text(
        json.dumps(models.config(16, 20, [layer])))
    with pytest.raises(ValueError):
        get_config(str(tmp_path))


@pytest.mark.parametrize("loop", [(0, 2, 2), (-1, 1, 2), (1, 0, 2)])
def test_loops_that_cannot_be(tmp_path, loop):
    (tmp_path / "config.json").write_text(json.dumps(
        models.config(16, 20, [models.mamba(8, 4, 2, 2)], loop)))
    with pytest.raises(ValueError, match="loop"):
        get_config(str(tmp_path))


def test_every_pass_has_a_cache_of_its_own(folder):
    cfg = get_config(folder("mixed")[0])
    kv = PagedKVCache(cfg, 1, 6, dtype=torch.bfloat16, state_slots=2)
    assert len(kv.layers) == 8
    held = [t for c in kv.layers for t in c]
    assert len({t.data_ptr() for t in held if t.numel()}) == \
        sum(t.numel() > 0 for t in held)
    looped = kv.layers[1], kv.layers[4]
    assert [t.shape for t in looped[0]] == [t.shape for t in looped[1]]
    # pages of keys and values, the convolution's last inputs, the delta
    # rule's state and its convolution's last inputs
    assert [t.dtype for t in looped[0]] == [
        torch.bfloat16, torch.bfloat16, torch.bfloat16, torch.float32,
        torch.bfloat16]


# ---- mechanisms alone -------------------------------------------------------

def rand(*shape, seed, scale=1.0):
    return scale * torch.randn(
        shape, generator=torch.Generator().manual_seed(seed))


def dtype_of(place):
    return getattr(torch, place[1])


def d64(t):
    return t.cpu().double()


def steps(place, cuts):
    """One request in portions: (rows, batch) of each, on pages in falling
    order and slot 1."""
    pages = list(range((sum(cuts) + 15) // 16))[::-1]
    at = 0
    for n in cuts:
        yield slice(at, at + n), StepBatch.build(
            [([0] * n, at, pages[:(at + n + 15) // 16], 1, [])], 16,
            torch.device(place[0]))
        at += n


def near(got, want, place, factor=1.0):
    assert float((d64(got) - want).abs().max()) < \
        factor * tol(place) * max(1.0, float(want.abs().max()))


@EVERY_PLACE
def test_layer_norm_and_the_start_of_a_pass(place):
    """Added to the residual ahead of a norm: what the layer before made, the
    scaled embedding, the pass's vector."""
    rows, width = 9, 40
    x, w, b, vec = rand(rows, width, seed=1) + 0.7, \
        1 + rand(width, seed=2), rand(width, seed=3), rand(width, seed=4)
    table = put(rand(20, width, seed=5), place)
    delta = put(rand(rows, width, seed=6), place)
    tok = torch.arange(rows, dtype=torch.int32) * 7 % 20
    dev = place[0]
    embedded = (tok.to(dev), table, 1.7)
    e = d64(table)[tok.long()] * 1.7
    for old, extra, t in ((x, delta, 2), (None, None, 0)):
        got_x, y = ops.add_norm(
            None if old is None else old.to(dev, copy=True), w.to(dev),
            b.to(dev), 1e-2, dtype_of(place), extra, None, embedded,
            vec.to(dev))
        want = e if old is None else old.double() + d64(extra)
        want = oracle.begin_pass({"loop.step": {t: vec.double()}}, want, e, t)
        assert got_x.dtype == torch.float32
        assert float((d64(got_x) - want).abs().max()) < 1e-5
        near(y, oracle.layer_norm(want, w, b, 1e-2), place)


@EVERY_PLACE
@CUTS
@pytest.mark.parametrize("taps,channels", [(4, 48), (1, 16), (3, 13), (6, 40)])
def test_short_convolution(place, cuts, taps, channels):
    n = sum(cuts)
    x = put(rand(n, channels, seed=1), place)
    w, b = rand(channels, taps, seed=2), rand(channels, seed=3)
    state = put(rand(3, taps - 1, channels, seed=4, scale=50.0), place)
    other = state[[0, 2]].clone()
    got = torch.cat([ops.short_conv(x[r], w.to(place[0]), b.to(place[0]),
                                    True, state, batch)
                     for r, batch in steps(place, cuts)])
    near(got, oracle.silu(oracle.short_conv(d64(x), w.double()) + b), place)
    assert torch.equal(state[1], x[n - taps + 1:])
    assert torch.equal(state[[0, 2]], other)


@EVERY_PLACE
@CUTS
@pytest.mark.parametrize("heads,kv,dim,dims,taps", [
    (4, 2, 24, 16, 4), (3, 3, 9, 6, 2), (2, 1, 64, 64, 1)])
def test_convolved_and_rotated_heads(place, cuts, heads, kv, dim, dims, taps):
    """Neighbouring elements turn together; values are the keys ahead of
    it."""
    n, rows = sum(cuts), (heads + kv) * dim
    buf = put(rand(n, rows + 5, seed=1), place)
    bias, w = rand(rows, seed=2), rand(rows, taps, seed=3)
    state = put(rand(3, taps - 1, rows, seed=4, scale=50.0), place)
    pages = (n + 15) // 16
    kc, vc = (torch.zeros(pages, kv, 16, dim, dtype=buf.dtype,
                          device=place[0]) for _ in range(2))
    rot = RotarySpec(50.0, dims, True)
    turns = rot.turns(place[0])
    q = torch.cat([ops.conv_rope(
        buf[r], bias.to(place[0]), w.to(place[0]), state,
        ops.rope_table(batch, rot, turns, {}), kc, vc, batch)
        for r, batch in steps(place, cuts)])
    u = d64(buf)[:, :rows] + bias
    if place[1] == "bfloat16":      # what is kept between steps is rounded
        u = u.bfloat16().double()
    c = oracle.short_conv(u, w.double())
    turned = oracle.rotate(c.view(n, heads + kv, dim), 50.0, dims)
    near(q, turned[:, :heads].reshape(n, -1), place)

    def held(cache):
        return cache.flip(0).transpose(1, 2).reshape(-1, kv, dim)[:n]
    near(held(kc), turned[:, heads:], place)
    near(held(vc), c[:, heads * dim:].view(n, kv, dim), place)


@EVERY_PLACE
def test_rotation_far_away(place):
    """Angles of positions beyond a million, whose products with frequencies
    32 bits cannot hold."""
    rot = RotarySpec(100.0, 16, True)
    batch, _ = request_batch(place, [(0, 2)])
    for p in (65536, 1000003, 16000001):
        batch.positions[:] = torch.tensor([p, p + 1])
        got = ops.rope_table(batch, rot, rot.turns(place[0]), {}).cpu()
        for r in (0, 1):
            for i in range(8):
                a = (p + r) * 100.0 ** (-2.0 * i / 16)
                assert abs(got[r, i, 0] - math.cos(a)) < 1e-5, (p, i)
                assert abs(got[r, i, 1] - math.sin(a)) < 1e-5, (p, i)


def window_case(place, spans, heads, kv, dim, sharp=1.0):
    batch, pages = request_batch(place, spans)
    q = put(rand(batch.tokens.shape[0], heads * dim, seed=1, scale=sharp),
            place)
    kc, vc = (put(rand(pages, kv, 16, dim, seed=s), place) for s in (2, 3))
    return batch, q, kc, vc


@EVERY_PLACE
@pytest.mark.parametrize("size,keep", [(24, 3), (16, 0), (1, 1), (17, 19),
                                       (500, 2), (5, 40)])
@pytest.mark.parametrize("heads,kv,dim,cap", [(4, 2, 24, 3.0), (3, 1, 9, 8.0),
                                              (2, 2, 64, 50.0)])
def test_window_attention(place, size, keep, heads, kv, dim, cap):
    spans = [(0, 2), (15, 1), (0, 1), (30, 37), (63, 2), (90, 1), (0, 33)]
    batch, q, kc, vc = window_case(place, spans, heads, kv, dim, 2.0)
    sink = rand(heads, seed=4, scale=1.5)
    got = ops.attn_ctx(q, None, kc, vc, None, batch, dim ** -0.5,
                       window=size, keep=keep, softcap=cap,
                       sink=sink.to(place[0]), mult=0.7)
    row = 0
    for e, i in enumerate(sorted(range(len(spans)),
                                 key=lambda i: spans[i][1] > 1)):
        first, n = spans[i]
        ids = batch.block_table[e, :(first + n + 15) // 16].long()
        k, v = (d64(c[ids]).transpose(1, 2).reshape(-1, kv, dim)[:first + n]
                for c in (kc, vc))
        qq = torch.zeros(first + n, heads, dim, dtype=torch.float64)
        qq[first:] = d64(q)[row:row + n].view(n, heads, dim)
        o = oracle.attend(qq, k, v, dim ** -0.5, cap, size, keep,
                          sink.double())
        near(got[row:row + n], 0.7 * o[first:].reshape(n, -1), place)
        row += n


@EVERY_PLACE
@pytest.mark.parametrize("size,keep", [(40, 4), (16, 0), (17, 33), (64, 1),
                                       (300, 0)])
@pytest.mark.parametrize("key", [0, 1, 3, 4, 15, 16, 32, 33, 63, 64, 300])
def test_a_key_that_stands_out(place, size, keep, key):
    """Found by every position that sees it and by no other: in prompts, in
    decoding, at the window's edge, among the first tokens, at page
    borders."""
    dim = 32
    edge = key + size
    spans = [(0, 140), (key, 2), (max(key - 1, 0), 3), (edge - 2, 2),
             (edge - 1, 3), (edge, 2)] + \
        [(p, 1) for p in sorted({key, key + 1, max(key - 1, 0), edge - 1,
                                 edge, edge + 1, 600})]
    for span in spans:
        batch, pages = request_batch(place, [span])
        n, length = batch.tokens.shape[0], span[0] + span[1]
        kc, vc = torch.zeros(2, pages, 1, 16, dim).unbind()
        for p in range(length):
            vc[batch.block_table[0, p // 16], 0, p % 16, p % dim] = 1.0
        if key < length:
            at = batch.block_table[0, key // 16], 0, key % 16
            kc[at][3] = 30.0
            vc[at].zero_()[5] = 7.0
        q = torch.zeros(n, dim)
        q[:, 3] = 1.0
        got = ops.attn_ctx(put(q, place), None, put(kc, place),
                           put(vc, place), None, batch, 1.0, window=size,
                           keep=keep, softcap=25.0,
                           sink=torch.zeros(1, device=place[0])).float().cpu()
        for row, p in zip(got, batch.positions.tolist()):
            if oracle.visible(p, key, size, keep):
                assert row[5] > 6.9, (p, key)
            else:
                seen = sum(oracle.visible(p, j, size, keep)
                           for j in range(p + 1))
                assert abs(float(row.sum()) - seen / (seen + 1)) < 1e-2, \
                    (p, key)


@EVERY_PLACE
@pytest.mark.parametrize("first", [0, 5, 100, 700])
def test_sinks_count_once(place, first):
    """With equal scores of zero a sink s leaves n / (n + e^s) of a value that
    is 1 everywhere, also where several workgroups share a context."""
    batch, pages = request_batch(place, [(first, 1), (first, 2)])
    kc, vc = (put(torch.full((pages, 2, 16, 16), float(i)), place)
              for i in (0, 1))
    q = put(torch.ones(3, 64), place)
    sink = torch.tensor([-3.0, 0.0, 4.0, 9.0])
    got = ops.attn_ctx(q, None, kc, vc, None, batch, 1.0, softcap=5.0,
                       sink=sink.to(place[0]))
    for row, p in zip(got.float().cpu(), batch.positions.tolist()):
        want = (p + 1) / (p + 1 + sink.exp())
        assert torch.allclose(row.view(4, 16), want[:, None].expand(4, 16),
                              atol=5e-3)


@EVERY_PLACE
@CUTS
@pytest.mark.parametrize("channels,n", [(48, 16), (13, 5), (40, 1), (32, 40)])
def test_selective_scan(place, cuts, channels, n):
    total = sum(cuts)
    u, gate = (put(rand(total, channels, seed=s), place) for s in (1, 2))
    z, zb = rand(total, channels, seed=3), rand(channels, seed=4) - 2
    low = put(rand(total, 3 + 2 * n, seed=5), place)
    a, d = -rand(channels, n, seed=6).exp(), rand(channels, seed=7)
    state = rand(3, channels, n, seed=8, scale=50.0).to(place[0])
    out = torch.empty_like(u)
    dev = [t.to(place[0]) for t in (z, zb, a, d)]
    for r, batch in steps(place, cuts):
        ops.selective_scan(u[r], gate[r], dev[0][r], dev[1], low[r], 3,
                           dev[2], dev[3], state, batch, out[r])
    x, bc = d64(u), d64(low)[:, 3:]
    y = oracle.selective_scan(x, oracle.softplus((z + zb).double()),
                              a.double(), bc[:, :n], bc[:, n:], d.double())
    near(out, y * oracle.silu(d64(gate)), place)


@EVERY_PLACE
@CUTS
@pytest.mark.parametrize("heads,dim,vdim,decay", [
    (2, 32, 16, [0.999, 0.2]), (3, 7, 11, [1.0, 0.9, 0.01]),
    (1, 128, 128, [0.97])])
def test_lightning_attention(place, cuts, heads, dim, vdim, decay):
    n, nq = sum(cuts), heads * dim
    x = put(rand(n, 2 * nq + heads * vdim + 3, seed=1), place)
    state = rand(3, heads, dim, vdim, seed=2, scale=50.0).to(place[0])
    dev = torch.tensor(decay, device=place[0])
    got = torch.cat([ops.lightning(x[r], dev, state, batch)
                     for r, batch in steps(place, cuts)])
    act = oracle.silu(d64(x))
    q, k, v = (act[:, a:b].view(n, heads, -1) for a, b in (
        (0, nq), (nq, 2 * nq), (2 * nq, 2 * nq + heads * vdim)))
    want = oracle.lightning_recurrence(q, k, v, decay)
    near(got, want.reshape(n, -1), place)


@EVERY_PLACE
def test_norm_over_all_heads_and_gate(place):
    o, gate = (put(rand(9, 77, seed=s), place) for s in (1, 2))
    norm = 1 + rand(77, seed=3)
    out = torch.empty_like(o)
    ops.joint_gate(o, norm.to(place[0]), gate, 1e-2, out)
    near(out, oracle.rms(d64(o), 1e-2) * norm * oracle.sigmoid(d64(gate)),
         place)


@EVERY_PLACE
@CUTS
@pytest.mark.parametrize("heads,kv,dim,vdim", [
    (4, 2, 16, 24), (3, 1, 7, 11), (1, 1, 128, 128), (2, 2, 64, 32)])
@pytest.mark.parametrize("zb", [-4.0, 4.0])
def test_delta_rule(place, cuts, heads, kv, dim, vdim, zb):
    """zb: slow and fast decays."""
    n, nq = sum(cuts), kv * dim
    qkv = put(rand(n, 2 * nq + heads * vdim, seed=1), place)
    z, bias = rand(n, heads * dim, seed=2, scale=2.0), \
        rand(heads * dim, seed=3) + zb
    rate, norm = rand(heads, seed=4).exp(), 1 + rand(vdim, seed=5)
    beta = put(rand(n, heads, seed=6, scale=2.0), place)
    gate = put(rand(n, heads * vdim, seed=7), place)
    state = rand(3, heads, dim, vdim, seed=8, scale=50.0).to(place[0])
    out = torch.empty_like(gate)
    dz, db, dr, dn = (t.to(place[0]) for t in (z, bias, rate, norm))
    for r, batch in steps(place, cuts):
        ops.delta(qkv[r], dz[r], db, dr, beta[r], dn, gate[r], state, batch,
                  kv, 1e-3, 0.6, out[r])
    x, per = d64(qkv), heads // kv
    q, k = (oracle.unit(x[:, a:a + nq].view(n, kv, dim))
            .repeat_interleave(per, 1) for a in (0, nq))
    g = torch.exp(-rate.double()[:, None] * oracle.softplus(
        (z + bias).double()).view(n, heads, dim))
    o = oracle.delta_recurrence(q * dim ** -0.5, k,
                                x[:, 2 * nq:].view(n, heads, vdim), g,
                                oracle.sigmoid(d64(beta)))
    want = 0.6 * (oracle.rms(o, 1e-3) * norm).reshape(n, -1) * \
        oracle.sigmoid(d64(gate))
    near(out, want, place, 2.0)


@EVERY_PLACE
def test_a_delta_rule_overwrites(place):
    """With full steps and no decay a key written twice holds its last value
    only."""
    n, dim, vdim = 40, 8, 4
    qkv = torch.zeros(n, 2 * dim + vdim)
    keys = torch.arange(n) % 3
    qkv[torch.arange(n), dim + keys] = 30.0
    qkv[torch.arange(n), keys] = 30.0
    qkv[:, 2 * dim:] = torch.arange(n)[:, None] % 7 - 3.0 + \
        torch.arange(vdim)
    dev = place[0]
    big = torch.full((n, 1), 40.0)
    out = torch.empty(n, vdim, dtype=dtype_of(place), device=dev)
    batch, _ = request_batch(place, [(0, n)])
    state = torch.zeros(1, 1, dim, vdim, device=dev)
    ops.delta(put(qkv, place), torch.full((n, dim), -60.0, device=dev),
              torch.zeros(dim, device=dev), torch.ones(1, device=dev),
              put(big, place), torch.ones(vdim, device=dev),
              put(big.expand(n, vdim).contiguous(), place), state, batch, 1,
              1e-5, 1.0, out)
    v = qkv[:, 2 * dim:].double()
    near(out, oracle.rms(v * dim ** -0.5, 1e-5), place)
    for k in range(3):
        near(state[0, 0, k], v[keys == k][-1], place)


@EVERY_PLACE
@pytest.mark.parametrize("experts,top", [(8, 3), (5, 5), (1, 1), (7, 2),
                                         (64, 8)])
@pytest.mark.parametrize("rows,width,ff,limit", [(1, 40, 24, 0.5),
                                                 (45, 19, 7, 2.0),
                                                 (33, 64, 64, 1.0)])
def test_experts(place, experts, top, rows, width, ff, limit):
    moe = MoESpec(experts, top, ff, glu=GluSpec("clamped", limit),
                  over_chosen=True, bias=True)
    y = put(rand(rows, width, seed=rows), place)
    router = put(rand(experts, width, seed=2, scale=2 * width ** -0.5), place)
    bias = rand(experts, seed=3)
    up = put(rand(experts, 2 * ff, width, seed=4, scale=2 * width ** -0.5),
             place)
    down = put(rand(experts, width, ff, seed=5, scale=ff ** -0.5), place)
    p = ops.experts(y, router, up, down, moe, bias.to(place[0]))
    got = (p.rows[p.at.long()].double() * p.weights[:, :, None]).sum(1)
    w = {"router": d64(router), "router.b": bias.double()}
    for e in range(experts):
        w[f"e{e}.gate"], w[f"e{e}.up"] = d64(up[e, 0::2]), d64(up[e, 1::2])
        w[f"e{e}.down"] = d64(down[e])
    near(got, oracle.experts(w, "", {"router": {"top": top}, "expert": {
        "limit": limit}}, d64(y)), place)


@EVERY_PLACE
@pytest.mark.parametrize("act,limit", [("relu", 0.0), ("clamped", 0.9)])
def test_gated_feed_forwards(place, act, limit):
    """Projections by identity matrices: only the gated product is left."""
    f = 40
    x = put(rand(9, 2 * f, seed=1, scale=2.0), place)
    out = torch.empty(9, f, dtype=x.dtype, device=place[0])
    ops.glu(x, GluSpec(act, limit), out)
    h, e = d64(x), torch.eye(2 * f, dtype=torch.float64)
    w = {"gate": e[:f], "up": e[f:], "down": e[:f, :f]}
    near(out, oracle.relu_glu(w, "", h) if act == "relu"
         else oracle.clamped_glu(w, "", h, limit), place)


@EVERY_PLACE
def test_logits_are_capped(place):
    x = put(rand(3, 101, seed=1, scale=30.0), place)
    want = oracle.softcap(d64(x), 12.0)
    near(ops.softcap(x, 12.0), want, place)


# ---- whole models -----------------------------------------------------------

@EVERY_PLACE
@pytest.mark.parametrize("name", list(models.CONFIGS))
def test_whole_prompts(folder, name, place):
    d, cfg, w = folder(name)
    for n, seed in ((130, 1), (1, 2), (2, 3), (17, 4)):
        toks = models.tokens(cfg, n, seed)
        want = expected(cfg, w, toks, (name, n, seed))
        replay_cut(d, place, toks, [n]).check("a", want)


@pytest.mark.parametrize("name", list(models.CONFIGS))
def test_residual_after_every_layer(folder, name, monkeypatch):
    """Not only the logits: what each layer leaves, in every pass."""
    d, cfg, w = folder(name)
    toks = models.tokens(cfg, 17, 4)
    streams = []
    oracle.forward(cfg, w, toks, streams)
    trace = TraceReplay(d, "float32", 64, "cpu")
    seen, whole = [], ops.add_norm

    def spy(x, w, b, eps, dtype, rows=None, picked=None, *rest):
        if x is not None:
            seen.append(whole(x.clone(), w, b, eps, dtype, rows, picked)[0])
        return whole(x, w, b, eps, dtype, rows, picked, *rest)
    monkeypatch.setattr(ops, "add_norm", spy)
    trace.step([{"id": "a", "tokens": toks, "want": list(range(17))}], [])
    assert len(seen) == len(streams)
    for got, want in zip(seen, streams):
        assert float((got - want).abs().max()) < 1e-4


@EVERY_PLACE
@pytest.mark.parametrize("name", list(models.CONFIGS))
def test_token_by_token(folder, name, place):
    """From the first token on, across page and window edges."""
    d, cfg, w = folder(name)
    toks = models.tokens(cfg, 130, 1)
    want = expected(cfg, w, toks, (name, 130, 1))
    replay_cut(d, place, toks, [1] * 130).check("a", want)


@EVERY_PLACE
@pytest.mark.parametrize("name", ["mixed", "odd", "large"])
@pytest.mark.parametrize("size", [2, 3, 7, 16, 17, 33, 64])
def test_portions(folder, name, size, place):
    d, cfg, w = folder(name)
    toks = models.tokens(cfg, 130, 1)
    want = expected(cfg, w, toks, (name, 130, 1))
    cuts = [size] * (110 // size)
    cuts += [110 - sum(cuts)] if sum(cuts) < 110 else []
    replay_cut(d, place, toks, cuts + [1] * 20).check("a", want)


@EVERY_PLACE
@pytest.mark.parametrize("name", ["mixed", "odd"])
def test_unequal_requests_in_one_batch(folder, name, place):
    """Portions beside single tokens, requests that pause, end and start, in
    a pool that makes them use each other's pages and slots."""
    d, cfg, w = folder(name)
    seeds = {"a": (130, 1), "b": (50, 5), "c": (90, 6), "d": (17, 4),
             "e": (60, 7), "f": (40, 8)}
    toks = {k: models.tokens(cfg, n, s) for k, (n, s) in seeds.items()}
    r = Replayed(d, place, 384)
    kv = r.trace.engine.kv
    free = kv.allocator.free_count, kv.slots.free_count

    def step(*parts, end=()):
        r.step([(k, toks[k], n) for k, n in parts], end)
    step(("a", 2), ("b", 31))
    step(("b", 1), ("a", 40), ("c", 3))
    step(("c", 1), ("b", 1), ("a", 1), ("d", 16))
    step(("d", 1), ("a", 50), ("b", 16), end=["d"])
    step(("b", 1), ("a", 1), end=["b"])
    step(("e", 60), ("c", 29), ("a", 1))
    step(("a", 1), ("f", 2))
    step(("f", 37), ("a", 20), ("c", 57), end=["c", "e"])
    step(("f", 1), ("a", 13), end=["a", "f"])
    for k, (n, s) in seeds.items():
        r.check(k, expected(cfg, w, toks[k], (name, n, s)))
    assert (kv.allocator.free_count, kv.slots.free_count) == free


@EVERY_PLACE
def test_pages_and_slots_are_used_again(folder, place):
    """One pool, one request after another in it: what the last one left
    must not show."""
    d, cfg, w = folder("mixed")
    r = Replayed(d, place, 192)
    for i, (n, seed) in enumerate([(130, 1), (17, 4), (90, 6), (130, 1),
                                   (2, 3)]):
        toks = models.tokens(cfg, n, seed)
        r.step([(f"r{i}", toks, n - 1)])
        r.step([(f"r{i}", toks, 1)], end=[f"r{i}"])
        r.check(f"r{i}", expected(cfg, w, toks, ("mixed", n, seed)))


@EVERY_PLACE
def test_only_wanted_rows_go_past_the_last_mixer(folder, place):
    d, cfg, w = folder("mixed")
    toks = models.tokens(cfg, 130, 1)
    want = expected(cfg, w, toks, ("mixed", 130, 1))
    trace = TraceReplay(d, place[1], 192, place[0])

    def step(a, n, wanted):
        return trace.step([{"id": "a", "tokens": toks[a:a + n],
                            "want": wanted}], [])
    assert step(0, 50, []).shape == (0, cfg["vocab"])
    assert error(step(50, 40, [39, 0, 7]), want[[89, 50, 57]]) < \
        LIMIT[place[1]]
    assert step(90, 1, []).shape == (0, cfg["vocab"])
    assert error(step(91, 1, [0]), want[[91]]) < LIMIT[place[1]]


def rotate_halves(x, base, dims):
    """Element i turns with element i + dims / 2."""
    pairs = [i // 2 + i % 2 * (dims // 2) for i in range(dims)]
    out = x.clone()
    out[..., pairs] = rotate(x[..., pairs], base, dims)
    return out


def delayed(u, taps):
    return short_conv(torch.cat([torch.zeros_like(u[:1]), u[:-1]]), taps)


def read_before_write(q, k, v, g, beta):
    n, heads, d = q.shape
    s = torch.zeros(heads, d, v.shape[2], dtype=q.dtype)
    out = torch.zeros_like(v)
    for t in range(n):
        s = g[t][..., None] * s
        out[t] = (s.transpose(1, 2) @ q[t][..., None])[..., 0]
        u = beta[t][:, None] * (v[t] - (s.transpose(1, 2)
                                        @ k[t][..., None])[..., 0])
        s = s + k[t][..., None] * u[:, None]
    return out


def first_pass_only(cfg):
    again = (cfg["loop"]["stop"] - cfg["loop"]["start"]) * \
        (cfg["loop"]["times"] - 1)
    runs, end = passes(cfg), cfg["loop"]["stop"]
    return runs[:end] + runs[end + again:]


rotate, short_conv, passes = oracle.rotate, oracle.short_conv, oracle.passes
clamped, route = oracle.clamped_glu, oracle.route
attend, mamba = oracle.attend, oracle.selective_scan
lightning = oracle.lightning_recurrence
PLANTED = {
    "window one longer": ("visible", lambda i, j, n, k:
                          j <= i and (i - j <= n or j < k)),
    "window one shorter": ("visible", lambda i, j, n, k:
                           j <= i and (i - j < n - 1 or j < k)),
    "nothing kept": ("visible", lambda i, j, n, k: j <= i and i - j < n),
    "one more kept": ("visible", lambda i, j, n, k:
                      j <= i and (i - j < n or j <= k)),
    "no sink": ("attend", lambda q, k, v, s, c, n, keep, sink: attend(
        q, k, v, s, c, n, keep, sink - 99)),
    "no caps": ("softcap", lambda z, cap: z),
    "halves rotated": ("rotate", rotate_halves),
    "positions counted from the end": ("rotate", lambda x, b, n:
                                       rotate(x.flip(0), b, n).flip(0)),
    "convolution a token late": ("short_conv", delayed),
    "no convolution": ("short_conv", lambda u, taps: u),
    "read before the write": ("delta_recurrence", read_before_write),
    "unit vectors forgotten": ("unit", lambda x: x),
    "no skip": ("selective_scan", lambda x, dt, a, b, c, d: mamba(
        x, dt, a, b, c, 0 * d)),
    "state not decayed": ("selective_scan", lambda x, dt, a, b, c, d: mamba(
        x, dt, 0 * a, b, c, d)),
    "constant decays": ("lightning_recurrence", lambda q, k, v, decay:
                        lightning(q, k, v, [0.9] * len(decay))),
    "mean kept": ("layer_norm", lambda x, w, b, eps:
                  oracle.rms(x, eps) * w + b),
    "no limits": ("clamped_glu", lambda w, p, h, limit:
                  clamped(w, p, h, 99.0)),
    "one expert more": ("route", lambda z, top:
                        route(z, min(top + 1, len(z)))),
    "no second pass": ("passes", first_pass_only),
    "embedding not added again": ("begin_pass", lambda w, x, e, t:
                                  x + w["loop.step"][t]),
    "no pass vectors": ("begin_pass", lambda w, x, e, t: x + (e if t else 0)),
}


@pytest.mark.parametrize("what", list(PLANTED))
def test_faults_would_show(folder, monkeypatch, what):
    """A mistake planted in the oracle is outside every limit above."""
    d, cfg, w = folder("mixed")
    toks = models.tokens(cfg, 130, 1)
    r = replay_cut(d, ("cpu", "float32"), toks, [130])
    monkeypatch.setattr(oracle, *PLANTED[what])
    wrong = oracle.forward(cfg, w, toks)
    assert error(torch.cat(r.got["a"]), wrong) > 2 * LIMIT["bfloat16"]


# ---- generation -------------------------------------------------------------

@EVERY_PLACE
@pytest.mark.parametrize("name", list(models.CONFIGS))
def test_greedy_generation(folder, name, place):
    """More requests than a batch holds, prompts longer than a step's
    tokens."""
    d, cfg, w = folder(name)
    lens, new = (70, 5, 100, 1, 33), (30, 12, 9, 40, 1)
    prompts = [models.tokens(cfg, n, 20 + n) for n in lens]
    eng = engine_for(d, place)
    got = generate(eng, prompts, new)
    for p, g, n in zip(prompts, got, new):
        assert len(g) == n
        same = check_greedy(cfg, w, p, g, place[1])
        assert same > (0.98 if place[1] == "float32" else 0.6)
    assert eng.kv.allocator.free_count >= 63     # a page for padded lanes


@EVERY_PLACE
def test_generation_with_preemption(folder, place):
    """Too few pages for all: the youngest gives its pages and slot back and
    is computed again."""
    d, cfg, w = folder("mixed")
    prompts = [models.tokens(cfg, n, 40 + n) for n in (40, 45, 50)]
    eng = engine_for(d, place, kv_blocks=13)
    seen = []
    whole = eng._preempt_youngest
    eng._preempt_youngest = lambda: (seen.append(1), whole())
    got = generate(eng, prompts, (40, 40, 40))
    assert seen
    for p, g in zip(prompts, got):
        check_greedy(cfg, w, p, g, place[1])


@EVERY_PLACE
def test_long_decoding(folder, place):
    d, cfg, w = folder("mixed")
    prompt = models.tokens(cfg, 3, 77)
    eng = engine_for(d, place, max_seq_len=320)
    (got,) = generate(eng, [prompt], (250,))
    check_greedy(cfg, w, prompt, got, place[1])


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["mixed", "large"])
def test_captured_decode_equals_eager(folder, name, dtype):
    """Replays between eager steps of joining requests, padded lanes beside
    live ones: the same tokens as without capture."""
    d, cfg, _ = folder(name)
    prompts = [models.tokens(cfg, n, 60 + n) for n in (20, 3, 50, 31, 9, 44)]
    new = (50, 20, 35, 8, 30, 25)
    runs = []
    for graphs in (False, True, True):
        eng = engine_for(d, ("cuda", dtype), max_batch=5, use_graphs=graphs)
        ids = [eng.add_request(p, max_new_tokens=n)
               for p, n in zip(prompts[:3], new)]
        out = {}
        for step in range(200):
            if step in (7, 8, 19):
                k = len(ids)
                ids.append(eng.add_request(prompts[k], max_new_tokens=new[k]))
            for o in eng.step():
                out.setdefault(o.seq_id, []).append(o.token)
            if step % 5 == 0:
                torch.cuda.synchronize()
            if not eng.has_work():
                break
        assert (eng.graph_runner is not None) == graphs
        runs.append([out[i] for i in ids])
    assert [len(r) for r in runs[0]] == list(new)
    assert runs[1] == runs[2]
    same = sum(a == b for x, y in zip(runs[0], runs[1])
               for a, b in zip(x, y)) / sum(new)
    assert same == 1.0 if dtype == "float32" else same > 0.5


# ---- entry points -----------------------------------------------------------

@EVERY_PLACE
def test_trace_run(folder, place, tmp_path):
    d, cfg, w = folder("mixed")
    r = subprocess.run(
        [os.path.join(ROOT, "bin", "trace_run"), "--model", d, "--dtype",
         place[1], "--out", str(tmp_path), "--max-tokens", "192", "--device",
         place[0]], input="\n".join(map(json.dumps, TRACE)) + "\n",
        capture_output=True, text=True, timeout=110)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [x for x in r.stdout.splitlines() if x.startswith("done")] == \
        ["done 0", "done 1", "done 2"]
    assert sorted(os.listdir(tmp_path)) == ["0.f32", "2.f32"]

    def rows(step):
        data = (tmp_path / f"{step}.f32").read_bytes()
        return torch.frombuffer(bytearray(data), dtype=torch.float32).view(
            -1, cfg["vocab"])
    a = oracle.forward(cfg, w, [1, 2, 3, 5, 6])
    b = oracle.forward(cfg, w, [4, 9])
    assert error(rows(0), torch.stack([a[0], a[2], b[0]])) < LIMIT[place[1]]
    assert error(rows(2), torch.stack([b[0], a[4]])) < LIMIT[place[1]]


def test_served_over_http(folder, monkeypatch):
    from fastapi.testclient import TestClient
    from substratus_amd.serve import server
    d, cfg, w = folder("mixed")
    monkeypatch.setenv("MODEL_DIR", d)
    monkeypatch.setenv("PARAMS_PATH", os.path.join(d, "none.json"))
    monkeypatch.setattr(torch.cuda, "is_available", lambda: False)
    app = server.create_app()
    assert app.state.engine.mcfg.family == "vurazen"
    prompt = models.tokens(cfg, 20, 5)
    with TestClient(app) as client:
        r = client.post("/v1/completions", json={
            "prompt": prompt, "max_tokens": 6, "temperature": 0.0})
        assert r.status_code == 200
        assert r.json()["usage"]["prompt_tokens"] == 20
    app.state.worker.stop()


def test_generate_command(folder):
    from typer.testing import CliRunner
    from substratus_amd.cli.main import app
    d, cfg, w = folder("mixed")
    prompt = models.tokens(cfg, 12, 9)
    r = CliRunner().invoke(app, [
        "generate", "--model", d, "--tokens", ",".join(map(str, prompt)),
        "--max-tokens", "8", "--dtype", "float32", "--device", "cpu"])
    assert r.exit_code == 0, r.output
    got = [int(t) for t in r.output.strip().splitlines()[-1].split(",")]
    assert check_greedy(cfg, w, prompt, got, "float32") == 1.0


def test_no_quantized_weights_or_caches(folder):
    for kw in ({"quant": "q4_0"}, {"kv_dtype": "fp8"}):
        with pytest.raises(ValueError):
            Engine(EngineConfig(model=folder("mixed")[0],
                                dtype=torch.float32, kv_blocks=8,
                                max_seq_len=64, **kw), device="cpu")


def test_loader_writes_a_registered_model(tmp_path):
    from substratus_amd.loader import model_loader
    d = model_loader.run(str(tmp_path), {"name": "vurazen-tiny"})
    cfg = get_config(d)
    assert cfg.name == "vurazen-tiny"
    eng = Engine(EngineConfig(model=d, dtype=torch.float32, max_batch=2,
                              max_seq_len=64, kv_blocks=8), device="cpu")
    assert load_weights(eng.model, eng.mcfg, d, eng.device, torch.float32)
    assert len(generate(eng, [[1, 2, 3]], [4])[0]) == 4
