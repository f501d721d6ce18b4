"""What tests of models through the engine share: places to run, requests with
known tokens, generation, comparison with an oracle's logits."""

import pytest
import torch

from substratus_amd.models.weights import load_weights
from substratus_amd.serve.batch import StepBatch
from substratus_amd.serve.engine import Engine, EngineConfig
from substratus_amd.serve.trace import TraceReplay

PLACES = [pytest.param(("cpu", "float32"), id="cpu"),
          pytest.param(("cuda", "float32"), id="gpu-f32",
                       marks=pytest.mark.gpu),
          pytest.param(("cuda", "bfloat16"), id="gpu-bf16",
                       marks=pytest.mark.gpu)]
# of logits, root mean square, relative to the logits' own
LIMIT = {"float32": 1e-4, "bfloat16": 0.06}


def written_models(tmp_path_factory, models):
    """name -> (folder, config, weights), written when first asked for"""
    made = {}

    def get(name):
        if name not in made:
            d = str(tmp_path_factory.mktemp(name))
            made[name] = (d, *models.write(d, name))
        return made[name]
    return get


def error(got, want):
    d = got.double() - want
    d = d - d.mean(-1, keepdim=True)
    return float((d.pow(2).mean(-1).sqrt() / want.std()).max())


class Replayed:
    """A TraceReplay with whole requests' tokens known ahead."""

    def __init__(self, folder, place, max_tokens):
        device, self.dtype = place
        self.trace = TraceReplay(folder, self.dtype, max_tokens, device)
        self.got, self.at = {}, {}

    def step(self, parts, end=()):
        """parts: (name, all tokens, how many of them next)"""
        entries = []
        for name, toks, n in parts:
            a = self.at.get(name, 0)
            entries.append({"id": name, "tokens": toks[a:a + n],
                            "want": list(range(n))})
            self.at[name] = a + n
        logits = self.trace.step(entries, list(end))
        for name, _, n in parts:
            self.got.setdefault(name, []).append(logits[:n])
            logits = logits[n:]
        assert logits.shape[0] == 0

    def check(self, name, want):
        got = torch.cat(self.got[name])
        assert error(got, want[:got.shape[0]]) < LIMIT[self.dtype], name


def replay_cut(folder, place, toks, cuts):
    r = Replayed(folder, place, (len(toks) + 63) // 64 * 64)
    for n in cuts:
        r.step([("a", toks, n)])
    assert r.at["a"] == len(toks)
    return r


def put(t, place):
    return t.to(place[0], getattr(torch, place[1]))


def request_batch(place, spans):
    """One request per (first position, tokens), on pages in falling order."""
    entries, top = [], sum((a + n + 15) // 16 for a, n in spans)
    pages = top
    for i, (a, n) in enumerate(spans):
        need = (a + n + 15) // 16
        entries.append(([0] * n, a, list(range(top - 1, top - 1 - need, -1)),
                        i, []))
        top -= need
    return StepBatch.build(entries, 16, torch.device(place[0])), pages


def tol(place):
    return 2e-4 if place[1] == "float32" else 2e-2


def engine_for(folder, place, **kw):
    args = dict(max_batch=3, max_seq_len=192, kv_blocks=64, prefill_chunk=48)
    args.update(kw)
    dtype = getattr(torch, place[1])
    eng = Engine(EngineConfig(model=folder, dtype=dtype, **args),
                 device=place[0])
    assert load_weights(eng.model, eng.mcfg, folder, eng.device, dtype)
    return eng


def generate(eng, prompts, new):
    ids = [eng.add_request(p, max_new_tokens=n) for p, n in zip(prompts, new)]
    out = {i: [] for i in ids}
    for _ in range(2000):
        if not eng.has_work():
            break
        for o in eng.step():
            assert o.error is None
            out[o.seq_id].append(o.token)
    assert not eng.has_work()
    return [out[i] for i in ids]


def greedy_share(logits, prompt, got, dtype):
    """Every token is the choice of the oracle's logits for what precedes it,
    up to ties within rounding; the share that are its very choice."""
    logits = logits[len(prompt) - 1:-1]
    slack = 4 * LIMIT[dtype] * float(logits.std())
    best = logits.max(-1).values
    mine = logits[torch.arange(len(got)), torch.tensor(got)]
    assert bool((best - mine <= slack).all())
    return float((logits.argmax(-1) == torch.tensor(got)).double().mean())


TRACE = [{"step": 0, "entries": [
             {"id": "a", "tokens": [1, 2, 3], "want": [0, 2]},
             {"id": "b", "tokens": [4], "want": [0]}], "end": []},
         {"step": 1, "entries": [{"id": "a", "tokens": [5], "want": []}],
          "end": ["b"]},
         {"step": 2, "entries": [{"id": "c", "tokens": [4, 9], "want": [0]},
                                 {"id": "a", "tokens": [6], "want": [0]}],
          "end": ["a", "c"]}]
