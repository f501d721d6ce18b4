"""Ditalorn models through the engine against the plain float64 implementation
in tests/oracles, on the CPU ops and on the GPU kernels."""

import json
import math
import os
import subprocess

import pytest
import torch

from oracles import ditalorn as oracle
from oracles import ditalorn_models as models
from oracles.harness import (LIMIT, PLACES, TRACE, Replayed, engine_for,
                             error, generate, greedy_share, put, replay_cut,
                             request_batch, tol, written_models)
from substratus_amd.models import get_config
from substratus_amd.models.layers import (AttentionSpec, GluSpec,
                                          LatentAttentionSpec, MoESpec,
                                          QueryTemperature)
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


# ---- configuration, registry, cache -----------------------------------------

def moe_spec(experts, top, ff, groups=1, keep=1):
    return MoESpec(experts, top, ff, groups, keep, GluSpec("silu"),
                   sigmoid=True, correction=True, group_best=2)


def test_config_is_read_from_the_folder(folder):
    cfg = get_config(folder("mixed")[0])
    assert cfg.family == "ditalorn" and cfg.num_layers == 6
    assert (cfg.hidden_size, cfg.vocab_size) == (80, 101)
    assert cfg.max_position_embeddings == 400 and cfg.learned_pos_emb
    assert cfg.embed_scale == 1.5 and cfg.norm_offset == 1.0
    assert cfg.pre_norm and cfg.tie_word_embeddings
    assert cfg.layers[0].mixer == AttentionSpec(
        4, 2, 24, 40, 1.2 * 24 ** -0.5, taps=3,
        temp=QueryTemperature(1.5, 16), v_norm=True, out_bias=True,
        falloff=True, sigmoid=True)
    assert cfg.layers[1].mixer == LatentAttentionSpec(
        3, 24, 0, 16, 40, 1.2 * 24 ** -0.5, None, head_gate=True, q_rank=56,
        window=24)
    assert cfg.layers[0].moe == moe_spec(9, 3, 40, 3, 2)
    assert cfg.layers[2].moe == moe_spec(4, 1, 56)
    assert cfg.layers[1].moe is None


def test_param_count_matches_the_weights(folder):
    for name in models.CONFIGS:
        d, _, w = folder(name)
        big = sum(t.numel() for t in w.values() if t.dim() == 2)
        assert get_config(d).param_count() == big


def test_registered_sizes():
    for name in ("ditalorn-tiny", "ditalorn-1b", "ditalorn-7b"):
        cfg = get_config(name)
        assert cfg.layers and cfg.param_count() > 0


@pytest.mark.parametrize("change", [
    {"type": "other"}, {"mlp": {"kind": "other"}},
    {"mixer": models.att(3, 2, 8, 8, 2)["mixer"]},
    {"mlp": models.moe({}, 9, 2, 8, (2, 1))["mlp"]},
    {"mlp": models.moe({}, 8, 3, 8, (4, 1))["mlp"]}])
def test_what_cannot_be_is_refused(tmp_path, change):
    doc = models.config(16, 20, [dict(models.att(2, 2, 8, 8, 2), **change)])
    (tmp_path / "config.json").write_text(json.dumps(doc))
    with pytest.raises(ValueError):
        get_config(str(tmp_path))


@pytest.mark.parametrize("make", [
    lambda: AttentionSpec(1, 1, 8, 8, 1.0, qk_norm=True, taps=2),
    lambda: AttentionSpec(1, 1, 8, 8, 1.0, v_norm=True),
    lambda: LatentAttentionSpec(1, 8, 0, 8, 8, 1.0, None, out_gate=True,
                                head_gate=True),
    lambda: LatentAttentionSpec(1, 8, 4, 8, 8, 1.0, None, q_rank=8),
    lambda: MoESpec(4, 1, 8, sigmoid=True, over_chosen=True)])
def test_mechanisms_that_do_not_go_together(make):
    with pytest.raises(ValueError):
        make()


def test_what_the_cache_holds(folder):
    cfg = get_config(folder("mixed")[0])
    kv = PagedKVCache(cfg, 1, 6, dtype=torch.bfloat16, state_slots=3)
    assert [tuple(t.shape) for t in kv.layers[0]] == [
        (6, 2, 16, 24), (6, 2, 16, 40), (3, 2, 4 * 24 + 2 * 24 + 2 * 40)]
    assert [tuple(t.shape) for t in kv.layers[1]] == [(6, 1, 16, 40)]
    assert {t.dtype for held in kv.layers for t in held} == {torch.bfloat16}
    assert kv.slots.num_slots == 3
    assert PagedKVCache(get_config(folder("large")[0]), 1, 6,
                        state_slots=3).slots.num_slots == 0


def test_no_position_past_the_table(folder):
    d, cfg, _ = folder("odd")
    eng = engine_for(d, ("cpu", "float32"), max_seq_len=1000)
    assert eng.cfg.max_seq_len == cfg["max_positions"]
    with pytest.raises(AssertionError):
        eng.add_request([1] * 300, max_new_tokens=2)
    trace = TraceReplay(d, "float32", 640, "cpu")
    with pytest.raises(ValueError):
        trace.step([{"id": "a", "tokens": [1] * 302, "want": []}], [])


# ---- mechanisms alone -------------------------------------------------------

def rand(*shape, seed, scale=1.0):
    return scale * torch.randn(
        shape, generator=torch.Generator().manual_seed(seed))


def d64(t):
    return t.cpu().double()


def near(got, want, place, factor=1.0):
    assert float((d64(got) - want).abs().max()) < \
        factor * tol(place) * max(1.0, float(want.abs().max()))


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


@EVERY_PLACE
@pytest.mark.parametrize("width", [64, 51])
def test_embedding_and_positions(place, width):
    table, pos = (put(rand(n, width, seed=n), place) for n in (20, 30))
    norm = rand(width, seed=1)
    batch, _ = request_batch(place, [(0, 5), (29, 1), (17, 3)])
    batch.tokens[:] = torch.arange(9) * 7 % 20
    x, y = ops.embed_norm(batch.tokens, table, norm.to(place[0]), 1.0, 1e-2,
                          2.5, pos, batch.positions)
    want = d64(table)[batch.tokens.cpu().long()] * 2.5 + \
        d64(pos)[batch.positions.cpu().long()]
    assert x.dtype == torch.float32
    assert float((d64(x) - want).abs().max()) < 1e-5
    near(y, oracle.norm(want, norm, 1e-2), place)


@EVERY_PLACE
@CUTS
@pytest.mark.parametrize("heads,kv,dim,vdim,taps,every", [
    (4, 2, 24, 40, 4, 7), (3, 3, 9, 7, 2, 16), (2, 1, 64, 64, 1, 1),
    (6, 1, 16, 300, 3, 33), (1, 2, 8, 130, 6, 1000), (2, 2, 6, 10, 3, 5)])
def test_convolved_heads(place, cuts, heads, kv, dim, vdim, taps, every):
    """Bias, convolution, query temperature, value norm, cache."""
    heads *= kv
    n, nq, rows = sum(cuts), heads * dim, (heads + kv) * dim + kv * vdim
    buf = put(rand(n, rows + 5, seed=1), place)
    bias, w = rand(rows, seed=2), rand(rows, taps, seed=3)
    state = put(rand(3, taps - 1, rows, seed=4, scale=50.0), place)
    other = state[[0, 2]].clone()
    pages = (n + 15) // 16
    kc, vc = (torch.zeros(pages, kv, 16, size, dtype=buf.dtype,
                          device=place[0]) for size in (dim, vdim))
    q = torch.cat([ops.conv_qkv(
        buf[r], bias.to(place[0]), w.to(place[0]), state, kc, vc, batch,
        QueryTemperature(0.7, every), 1e-2) for r, batch in steps(place, cuts)])
    c = oracle.short_conv(d64(buf)[:, :rows] + bias, w.double())
    t = torch.tensor([oracle.temperature(p, 0.7, every) for p in range(n)])
    near(q, c[:, :nq] * t[:, None], place)

    def held(cache):
        return cache.flip(0).transpose(1, 2).reshape(-1, *cache.shape[1::2])[
            :n]
    near(held(kc), c[:, nq:nq + kv * dim].view(n, kv, dim), place)
    near(held(vc), oracle.value_norm(c[:, nq + kv * dim:].view(n, kv, vdim),
                                     1e-2), place)
    assert torch.equal(state[1], buf[n - taps + 1:, :rows])
    assert torch.equal(state[[0, 2]], other)


@EVERY_PLACE
def test_query_temperature_steps(place):
    """At the last position of a step and the first of the next, far away as
    near by."""
    for every in (1, 3, 64, 1000):
        for p in (0, every - 2, every - 1, every, 5 * every - 2,
                  5 * every - 1, 4097, 1000000):
            if p < 0:
                continue
            batch, _ = request_batch(place, [(0, 1)])
            batch.positions[:] = p
            buf = put(torch.ones(1, 24), place)
            kc, vc = (torch.zeros(1, 1, 16, 8, dtype=buf.dtype,
                                  device=place[0]) for _ in range(2))
            q = ops.conv_qkv(
                buf, None, torch.ones(24, 1, device=place[0]),
                torch.zeros(1, 0, 24, dtype=buf.dtype, device=place[0]), kc,
                vc, batch, QueryTemperature(0.5, every), 1e-5)
            want = 1 + 0.5 * math.log(math.floor((p + 1) / every) + 1)
            near(q, torch.full((1, 8), want, dtype=torch.float64), place, 0.2)


def sigmoid_case(place, spans, heads, kv, dim, vdim, sharp=1.0):
    batch, pages = request_batch(place, spans)
    q = put(rand(batch.tokens.shape[0], heads * dim, seed=1, scale=sharp),
            place)
    kc, vc = (put(rand(pages, kv, 16, size, seed=s), place)
              for s, size in ((2, dim), (3, vdim)))
    return batch, q, kc, vc


def requests(batch, spans):
    """(entry, first position, tokens) in the order of the batch's rows."""
    for e, i in enumerate(sorted(range(len(spans)),
                                 key=lambda i: spans[i][1] > 1)):
        yield e, *spans[i]


def held_rows(cache, batch, e, length):
    ids = batch.block_table[e, :(length + 15) // 16].long()
    c = d64(cache[ids]).transpose(1, 2)
    return c.reshape(-1, *c.shape[2:])[:length]


@EVERY_PLACE
@pytest.mark.parametrize("heads,kv,dim,vdim", [
    (4, 2, 24, 40), (3, 1, 9, 7), (7, 1, 56, 72), (2, 2, 128, 128),
    (5, 5, 16, 200)])
@pytest.mark.parametrize("steep", [0.0, 1.0])
def test_sigmoid_attention(place, heads, kv, dim, vdim, steep):
    spans = [(0, 2), (15, 1), (0, 1), (30, 37), (63, 2), (190, 1), (0, 133)]
    batch, q, kc, vc = sigmoid_case(place, spans, heads, kv, dim, vdim, 2.0)
    r1, r2 = steep * rand(heads, seed=4).abs(), rand(heads, seed=5).abs()
    pb = rand(heads, seed=6) - 2
    got = ops.attn_ctx(
        q, None, kc, vc, None, batch, dim ** -0.5,
        falloff=(r1.to(place[0]), r2.to(place[0])),
        weight_bias=pb.to(place[0]))
    row = 0
    for e, first, n in requests(batch, spans):
        k, v = (held_rows(c, batch, e, first + n) for c in (kc, vc))
        qq = torch.zeros(first + n, heads, dim, dtype=torch.float64)
        qq[first:] = d64(q)[row:row + n].view(n, heads, dim)
        o = oracle.attend_sigmoid(qq, k, v, dim ** -0.5, r1, r2, pb.double())
        near(got[row:row + n], o[first:].reshape(n, -1), place)
        row += n


@EVERY_PLACE
@pytest.mark.parametrize("key", [0, 1, 15, 16, 17, 63, 64, 300, 1023])
def test_a_key_that_stands_out(place, key):
    """Its value comes through alone, at the weight of its score and distance,
    at every later position, in prompts and in decoding; at none before."""
    dim, r1, r2, pb = 32, 1.3, 0.4, -24.0
    spans = [(0, 140), (key, 2), (max(key - 1, 0), 3), (key + 1, 40)] + \
        [(p, 1) for p in sorted({key, key + 1, max(key - 1, 0), 1500,
                                 (key // 16 + 1) * 16})]
    for span in spans:
        batch, pages = request_batch(place, [span])
        n = batch.tokens.shape[0]
        kc, vc = torch.zeros(2, pages, 1, 16, dim).unbind()
        vc[..., 7] = 1.0
        if key < span[0] + span[1]:
            at = batch.block_table[0, key // 16], 0, key % 16
            kc[at][3], vc[at][7], vc[at][5] = 30.0, 0.0, 2.0
        q = torch.zeros(n, dim)
        q[:, 3] = 1.0
        one = torch.ones(1, device=place[0])
        got = ops.attn_ctx(put(q, place), None, put(kc, place),
                           put(vc, place), None, batch, 1.0,
                           falloff=(one * r1, one * r2),
                           weight_bias=one * pb).float().cpu()
        for row, p in zip(got, batch.positions.tolist()):
            want = 0.0 if p < key else 2 / (1 + math.exp(-(
                30 + pb - r1 * math.log(1 + r2 * (p - key)))))
            assert abs(float(row[5]) - want) < 5 * tol(place), (p, key)
            assert abs(float(row[7])) < 1e-6


@EVERY_PLACE
@pytest.mark.parametrize("first", [0, 5, 100, 900, 3000])
def test_sigmoid_weights_add_up(place, first):
    """Equal scores of zero and a value that is 1 everywhere: the sum of all
    weights, also where several workgroups share a context."""
    batch, pages = request_batch(place, [(first, 1), (first, 2)])
    kc, vc = (put(torch.full((pages, 2, 16, 16), float(i)), place)
              for i in (0, 1))
    q = put(torch.ones(3, 64), place)
    pb, r1, r2 = torch.tensor([-6.0, -5.0, -3.0, 0.0]), \
        torch.tensor([0.0, 0.1, 1.0, 2.0]), torch.tensor([1.0, 3.0, 0.2, 1.0])
    got = ops.attn_ctx(q, None, kc, vc, None, batch, 1.0, falloff=(
        r1.to(place[0]), r2.to(place[0])), weight_bias=pb.to(place[0]))
    for row, p in zip(got.float().cpu(), batch.positions.tolist()):
        dist = torch.arange(p + 1).double()
        want = torch.sigmoid(pb[:, None] - r1[:, None] * torch.log(
            1 + r2[:, None] * dist)).sum(1)
        assert torch.allclose(row.view(4, 16).double(),
                              want[:, None].expand(4, 16), rtol=8e-3)


def spec_of(heads, dim, vdim, rank, window, scale=1.0, **kw):
    return LatentAttentionSpec(heads, dim, 0, vdim, rank, scale, None,
                               head_gate=True, q_rank=8, window=window, **kw)


def run_latent(spec, batch, q, gate, w, cache, expand=None):
    uk_t = w[:spec.heads * spec.dim].view(
        spec.heads, spec.dim, spec.rank).transpose(1, 2).contiguous()
    return ops.latent_attn(q, gate, cache, w, uk_t, batch, spec, {}, expand)


@EVERY_PLACE
@pytest.mark.parametrize("size", [1, 5, 16, 24, 64, 100, 500])
@pytest.mark.parametrize("heads,dim,vdim,rank", [
    (3, 24, 16, 40), (2, 9, 7, 21), (20, 16, 32, 64), (4, 64, 128, 512)])
@pytest.mark.parametrize("expand", [True, False])
def test_windowed_latent_attention(place, size, heads, dim, vdim, rank,
                                   expand):
    spec = spec_of(heads, dim, vdim, rank, size, 0.5)
    spans = [(0, 2), (15, 1), (16, 1), (30, 37), (90, 33), (63, 2), (0, 1),
             (150, 1), (0, 90)]
    batch, pages = request_batch(place, spans)
    n = batch.tokens.shape[0]
    q = put(rand(n, heads * dim, seed=1, scale=2.0), place)
    gate = put(rand(n, heads + 3, seed=2, scale=2.0), place)[:, 1:heads + 1]
    w = put(rand(heads * (dim + vdim), rank, seed=3, scale=rank ** -0.5),
            place)
    cache = put(rand(pages, 1, 16, rank, seed=4), place)
    got = run_latent(spec, batch, q, gate, w, cache, expand)
    row = 0
    for e, first, n in requests(batch, spans):
        c = held_rows(cache, batch, e, first + n)[:, 0]
        k = (c @ d64(w)[:heads * dim].T).view(-1, heads, dim)
        v = (c @ d64(w)[heads * dim:].T).view(-1, heads, vdim)
        qq = torch.zeros(first + n, heads, dim, dtype=torch.float64)
        qq[first:] = d64(q)[row:row + n].view(n, heads, dim)
        o = oracle.attend(qq, k, v, 0.5, size)[first:] * oracle.sigmoid(
            d64(gate)[row:row + n])[:, :, None]
        near(got[row:row + n], o.reshape(n, -1), place)
        row += n


@EVERY_PLACE
@pytest.mark.parametrize("size", [16, 40, 63, 64, 65, 300])
@pytest.mark.parametrize("key", [0, 1, 15, 16, 33, 63, 64, 300])
@pytest.mark.parametrize("expand", [True, False])
def test_a_key_at_the_window_s_edge(place, size, key, expand):
    """Found by every position that sees it and by no other: in prompts, in
    decoding, first and last of a window, at page borders."""
    dim, vdim, rank = 16, 24, 32
    spec = spec_of(1, dim, vdim, rank, size)
    w = torch.zeros(dim + vdim, rank)
    w[:dim, :dim] = torch.eye(dim)          # keys: the latents' beginning
    w[dim:dim + rank - dim, dim:] = torch.eye(rank - dim)   # values: its rest
    edge = key + size
    spans = [(0, 140), (key, 2), (max(key - 1, 0), 3), (edge - 2, 2),
             (edge - 1, 3), (edge, 2)] + \
        [(p, 1) for p in sorted({key, key + 1, max(key - 1, 0), edge - 1,
                                 edge, edge + 1, 600})]
    for span in spans:
        batch, pages = request_batch(place, [span])
        n, length = batch.tokens.shape[0], span[0] + span[1]
        cache = torch.zeros(pages, 1, 16, rank)
        cache[..., dim + 2] = 1.0
        if key < length:
            at = cache[batch.block_table[0, key // 16], 0, key % 16]
            at[3], at[dim + 2], at[dim + 5] = 30.0, 0.0, 7.0
        q = torch.zeros(n, dim)
        q[:, 3] = 1.0
        got = run_latent(spec, batch, put(q, place), None, put(w, place),
                         put(cache, place), expand).float().cpu()
        for row, p in zip(got, batch.positions.tolist()):
            seen = oracle.windowed(p, key, size)
            assert abs(float(row[5]) - 7.0 * seen) < 2e-2, (p, key)
            assert abs(float(row[2]) - (not seen)) < 1e-2, (p, key)


@EVERY_PLACE
@pytest.mark.parametrize("q_rank,rank,heads", [(56, 40, 3), (13, 21, 1),
                                               (300, 512, 8)])
def test_latents_of_queries_and_keys(place, q_rank, rank, heads):
    """Both normed, one in place, one into the cache; what follows them in a
    row is left alone."""
    n = 70
    buf = put(rand(n, q_rank + rank + heads, seed=1), place)
    qn, cn = 1 + 0.3 * rand(q_rank, seed=2), 1 + 0.3 * rand(rank, seed=3)
    batch, pages = request_batch(place, [(0, n)])
    cache = torch.zeros(pages, 1, 16, rank, dtype=buf.dtype, device=place[0])
    ref = d64(buf)
    spec = LatentAttentionSpec(heads, 8, 0, 8, rank, 1.0, None, q_rank=q_rank)
    ops.latent_prepare(buf, spec, q_rank, cn.to(place[0]), 1e-2,
                       torch.empty(0, dtype=torch.float64, device=place[0]),
                       batch.positions, cache, batch.slots, qn.to(place[0]))
    near(buf[:, :q_rank], oracle.rms(ref[:, :q_rank], 1e-2) * qn, place)
    near(held_rows(cache, batch, 0, n)[:, 0],
         oracle.rms(ref[:, q_rank:q_rank + rank], 1e-2) * cn, place)
    assert torch.equal(d64(buf)[:, q_rank:], ref[:, q_rank:])


@EVERY_PLACE
@pytest.mark.parametrize("experts,top,groups", [
    (12, 3, (3, 2)), (6, 2, (3, 1)), (5, 5, (5, 5)), (7, 3, None), (1, 1, None),
    (64, 8, (8, 4)), (130, 4, (13, 3)), (5, 2, (5, 3))])
@pytest.mark.parametrize("shift", [0.0, -2.0])
def test_routing(place, experts, top, groups, shift):
    """Corrections decide who is chosen, not the weights; a group counts by
    its two best; shift -2: all choice scores are negative."""
    z = 2 * rand(40, experts, seed=experts)
    corr = 0.5 * rand(experts, seed=experts + 1) + shift
    count, keep = groups or (1, 1)
    if place[0] == "cpu":
        from substratus_amd.ops import ref
        ids, wt = ref.moe_select(z, top, count, keep, False, True, corr, 2)
    else:
        ids = torch.empty(40, top, dtype=torch.int32, device="cuda")
        wt = torch.empty(40, top, device="cuda")
        ops._ext().moe_select(ids, wt, z.cuda()[None], count, keep, None,
                              False, True, corr.cuda(), 2)
    router = {"top": top}
    if groups:
        router["groups"] = {"count": count, "keep": keep}
    for t in range(40):
        want = oracle.route(z[t].double(), corr.double(), router)
        got = dict(zip(ids[t].tolist(), wt[t].tolist()))
        assert got.keys() == want.keys()
        assert all(abs(got[e] - float(want[e])) < 1e-6 for e in want)


@EVERY_PLACE
@pytest.mark.parametrize("rows", [1, 2, 45])
@pytest.mark.parametrize("width,moe", [
    (40, moe_spec(12, 3, 24, 3, 2)), (19, moe_spec(5, 2, 7)),
    (64, moe_spec(1, 1, 64))])
def test_experts(place, rows, width, moe):
    def weight(*s, seed):
        return put(rand(*s, seed=seed, scale=1.5 * s[-1] ** -0.5), place)
    y = put(rand(rows, width, seed=rows), place)
    router, up, down = weight(moe.experts, width, seed=1), \
        weight(moe.experts, 2 * moe.ff, width, seed=2), \
        weight(moe.experts, width, moe.ff, seed=3)
    corr = rand(moe.experts, seed=4) - 2
    p = ops.experts(y, router, up, down, moe, None, corr.to(place[0]))
    got = (p.rows[p.at.long()].double() * p.weights[:, :, None]).sum(1)
    w = {"router": d64(router), "correction": corr.double()}
    for e in range(moe.experts):
        w[f"e{e}.gate"], w[f"e{e}.up"] = d64(up[e])[::2], d64(up[e])[1::2]
        w[f"e{e}.down"] = d64(down[e])
    want = oracle.experts(w, "", {"top": moe.top, "groups": {
        "count": moe.groups, "keep": moe.keep}}, d64(y))
    assert float((got.cpu() - want).abs().max() / want.abs().max()) < \
        tol(place)


# ---- whole models -----------------------------------------------------------

@EVERY_PLACE
@pytest.mark.parametrize("name", list(models.CONFIGS))
def test_whole_prompts(folder, name, place):
    d, cfg, w = folder(name)
    for n, seed in ((130, 1), (1, 2), (2, 3), (17, 4)):
        toks = models.tokens(cfg, n, seed)
        want = expected(cfg, w, toks, (name, n, seed))
        replay_cut(d, place, toks, [n]).check("a", want)


def test_residual_after_every_layer(folder):
    """Not only the logits: what each layer leaves."""
    d, cfg, w = folder("mixed")
    toks = models.tokens(cfg, 17, 4)
    streams = []
    oracle.forward(cfg, w, toks, streams)
    trace = TraceReplay(d, "float32", 64, "cpu")
    seen, layers = [], trace.engine.model.layers
    whole = ops.stream_norm

    def spy(delta, x, *args, **kw):
        y = whole(delta, x, *args, **kw)
        seen.append(x.clone())
        return y
    ops.stream_norm = spy
    try:
        trace.step([{"id": "a", "tokens": toks, "want": list(range(17))}], [])
    finally:
        ops.stream_norm = whole
    at = -1
    for layer, want in zip(layers, streams):
        at += 2 if layer.spec.moe else 1
        assert float((seen[at] - want).abs().max()) < 1e-4
    assert at + 1 == len(seen)


@EVERY_PLACE
@pytest.mark.parametrize("name", list(models.CONFIGS))
def test_token_by_token(folder, name, place):
    """From the first token on, across page and window edges."""
    d, cfg, w = folder(name)
    toks = models.tokens(cfg, 130, 1)
    want = expected(cfg, w, toks, (name, 130, 1))
    replay_cut(d, place, toks, [1] * 130).check("a", want)


@EVERY_PLACE
@pytest.mark.parametrize("name", ["mixed", "odd", "large", "heads"])
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
    free = r.trace.engine.kv.allocator.free_count

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
    assert r.trace.engine.kv.allocator.free_count == free
    assert r.trace.engine.kv.slots.free_count == 4


@EVERY_PLACE
def test_pages_and_slots_are_used_again(folder, place):
    """One pool, one request after another in it: what the last one left
    must not show."""
    d, cfg, w = folder("mixed")
    r = Replayed(d, place, 192)
    for i, (n, seed) in enumerate([(130, 1), (17, 4), (90, 6), (130, 1),
                                   (2, 3), (1, 2), (17, 4)]):
        toks = models.tokens(cfg, n, seed)
        if n > 1:
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


route, temperature, windowed = oracle.route, oracle.temperature, \
    oracle.windowed
PLANTED = {
    "own key unseen": ("causal", lambda i, j: j < i or i == 0 == j),
    "one key ahead": ("causal", lambda i, j: j <= i + 1),
    "first key unseen": ("causal", lambda i, j: j <= i and (j or not i)),
    "window one wider": ("windowed", lambda i, j, s: windowed(i, j, s + 1)),
    "window one narrower": ("windowed", lambda i, j, s: windowed(
        i, j, max(s - 1, 1))),
    "no window": ("windowed", lambda i, j, s: j <= i),
    "no falloff": ("distance_penalty", lambda n, r1, r2: 0.0),
    "falloff by another base": ("distance_penalty", lambda n, r1, r2:
                                r1 * math.log2(1 + r2 * n)),
    "falloff one further": ("distance_penalty", lambda n, r1, r2:
                            r1 * math.log(1 + r2 * (n + 1))),
    "no temperature": ("temperature", lambda p, c, e: 1.0),
    "temperature one late": ("temperature", lambda p, c, e: temperature(
        max(p - 1, 0), c, e)),
    "temperature not floored": ("temperature", lambda p, c, e: 1 + c *
                                math.log((p + 1) / e + 1)),
    "values not normed": ("value_norm", lambda v, eps: v),
    "convolution turned round": ("short_conv", lambda u, t, conv=oracle
                                 .short_conv: conv(u, t.flip(1))),
    "no position vector": ("embed", lambda w, toks, s: w["embed"][toks] * s),
    "positions scaled": ("embed", lambda w, toks, s: s * (
        w["embed"][toks] + w["pos"][:len(toks)])),
    "norm weights as they are": ("norm", lambda x, w, eps:
                                 oracle.rms(x, eps) * w),
    "groups forgotten": ("route", lambda z, c, r: route(
        z, c, {"top": r["top"]})),
    "a group's best alone": ("group_score", max),
    "no correction": ("route", lambda z, c, r: route(z, 0 * c, r)),
    "one expert more": ("route", lambda z, c, r: route(
        z, c, dict(r, top=min(r["top"] + 1, len(z))))),
    "weights corrected": ("route", lambda z, c, r: {
        e: s + c[e] for e, s in route(z, c, r).items()}),
    "no gate": ("head_gate", lambda w, pre, h: torch.ones(
        h.shape[0], w[pre + "g"].shape[0], dtype=h.dtype)),
    "queries' latent not normed": ("query_latent", lambda w, pre, h, eps:
                                   h @ w[pre + "dq"].T * w[pre + "dq.norm"]),
    "latent not normed": ("latent", lambda w, pre, h, eps:
                          h @ w[pre + "dkv"].T * w[pre + "dkv.norm"]),
    "experts linear": ("silu", lambda z: z),
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
    """Too few pages for all: the youngest gives its pages and its slot back
    and is computed again."""
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
@pytest.mark.parametrize("name", ["mixed", "large", "heads"])
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
    assert app.state.engine.mcfg.family == "ditalorn"
    prompt = models.tokens(cfg, 20, 5)
    with TestClient(app) as client:
        r = client.post("/v1/completions", json={
            "prompt": prompt, "max_tokens": 6, "temperature": 0.0})
        assert r.status_code == 200
        assert r.json()["usage"]["prompt_tokens"] == 20
    app.state.worker.stop()


def test_generate_command(folder, monkeypatch):
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
    d = model_loader.run(str(tmp_path), {"name": "ditalorn-tiny"})
    cfg = get_config(d)
    assert cfg.name == "ditalorn-tiny"
    eng = Engine(EngineConfig(model=d, dtype=torch.float32, max_batch=2,
                              max_seq_len=64, kv_blocks=8), device="cpu")
    assert load_weights(eng.model, eng.mcfg, d, eng.device, torch.float32)
    assert len(generate(eng, [[1, 2, 3]], [4])[0]) == 4
