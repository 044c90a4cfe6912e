"""Bitatar through the framework — loader, cache, slots, batches, scheduler,
generation, command line — against the plain oracle.  On the CPU the reference
path runs; the GPU runs (marked) take the HIP kernels, in f32 and bf16."""
import json
import os
import subprocess
import sys

import pytest
import torch

from rbg_amd.engine.config import EngineConfig
from rbg_amd.engine.engine import LLMEngine
from rbg_amd.engine.kv_cache import BlockTable, OutOfPages
from rbg_amd.engine.sequence import SamplingParams
from rbg_amd.engine.trace import TraceSession
from rbg_amd.models.registry import load_config, resolve_model
from tests import bitatar_cases as cases
from tests.bitatar_cases import (answers, delta, latent, prompt, rel_err,
                                 row_errs)

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
GPU = pytest.mark.gpu
WHERE = [pytest.param(("cpu", "float32"), id="cpu-f32"),
         pytest.param(("cuda", "float32"), id="gpu-f32", marks=GPU),
         pytest.param(("cuda", "bfloat16"), id="gpu-bf16", marks=GPU)]
# positions, relative to the answers' RMS: almost all of them, and the worst.
# bf16's rounding is magnified where a head's output almost cancels before its
# norm, so the worst one has room; f32 has none.
TOL = {"float32": (3e-5, 3e-5), "bfloat16": (4e-2, 0.2)}

MODELS = {
    # every branch: unequal windows and ranks, a layer without feed-forward
    "mix": cases.config([delta(), latent(window=21),
                         latent(heads=2, dim=16, vdim=8, rank=16, window=5,
                                ff=None),
                         delta(heads=3, dim=16, ff=24)]),
    # sizes that no vector access divides, one group, two taps
    "odd": cases.config([latent(heads=1, dim=5, vdim=7, rank=11, window=9,
                                ff=21), delta(heads=1, dim=9, ff=None)],
                        width=35, vocab=67, groups=1, taps=2, eps=1e-3,
                        scale=1.0),
    # window of one token; five taps; recurrent first and last
    "edge": cases.config([delta(dim=32), latent(window=1),
                          latent(window=17, dim=32, vdim=32, rank=64),
                          delta(dim=32)], width=64, groups=4, taps=5),
    # no attention at all: pages of no size
    "rec": cases.config([delta(heads=2, dim=16)], taps=1),
}


@pytest.fixture(scope="module")
def model(tmp_path_factory):
    """name -> (folder, config, weights)"""
    made = {}

    def get(name):
        if name not in made:
            cfg = MODELS[name]
            w = cases.weights(cfg, seed=len(name))
            folder = cases.save(tmp_path_factory.mktemp(name), cfg, w)
            made[name] = (folder, cfg, w)
        return made[name]
    return get


_answers = {}


def want_of(model, name, n, seed=0):
    key = (name, n, seed)
    if key not in _answers:
        _, cfg, w = model(name)
        toks = prompt(n, cfg["vocab"], seed)
        _answers[key] = (toks, answers(toks, cfg, w))
    return _answers[key]


def session(folder, where, max_tokens, **kw):
    cfg = load_config(folder)
    cfg.dtype = where[1]
    return TraceSession(cfg, max_tokens, device=where[0], **kw)


def feed(s, rid, toks, want=True):
    return {"id": rid, "tokens": toks,
            "want": list(range(len(toks))) if want else []}


def check(got, want, where):
    err = row_errs(got, want).sort().values
    most, worst = TOL[where[1]]
    assert err[-1] < worst, err[-1]
    assert err[:max(1, int(0.95 * len(err)))][-1] < most or len(err) < 20, err


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("name", MODELS)
def test_whole_prompt_then_token_by_token(model, where, name):
    """One portion; the same token by token from an empty sequence; and a
    long decode after a short portion."""
    folder = model(name)[0]
    toks, want = want_of(model, name, 75)
    s = session(folder, where, 80)
    check(s.step([feed(s, "a", toks)], ["a"]), want, where)
    # the freed slot and pages serve the next request
    rows = [s.step([feed(s, "b", [t])], []) for t in toks]
    check(torch.cat(rows), want, where)
    s.step([], ["b"])
    rows = [s.step([feed(s, "c", toks[:3])], [])]
    rows += [s.step([feed(s, "c", [t])], []) for t in toks[3:]]
    check(torch.cat(rows), want, where)


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("name,sizes", [
    ("mix", [2]), ("mix", [3, 16, 1, 2, 33]), ("odd", [2, 5]),
    ("edge", [17, 2, 15, 1]), ("rec", [2, 3])])
def test_portions(model, where, name, sizes):
    """Cut anywhere: inside pages, windows and chunks, down to two tokens."""
    folder = model(name)[0]
    toks, want = want_of(model, name, 75)
    s = session(folder, where, 80)
    rows, at, i = [], 0, 0
    while at < len(toks):
        n = min(sizes[i % len(sizes)], len(toks) - at)
        rows.append(s.step([feed(s, 0, toks[at:at + n])], []))
        at, i = at + n, i + 1
    check(torch.cat(rows), want, where)


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("name", ["mix", "odd", "edge"])
def test_mixed_batches_reuse_pages_and_slots(model, where, name):
    """Unequal requests in every phase together, with barely enough pages and
    two slots fewer than requests; one pauses and goes on."""
    folder = model(name)[0]
    lens = {"a": 75, "b": 20, "c": 1, "d": 41, "e": 33, "f": 18}
    seqs = {k: want_of(model, name, n, seed=i)
            for i, (k, n) in enumerate(lens.items())}
    s = session(folder, where, 208, max_requests=4)
    at, got, done = dict.fromkeys(lens, 0), {k: [] for k in lens}, set()
    waiting, live = list(lens), []
    portions = [1, 9, 2, 17, 1, 1, 30]
    step = 0
    while len(done) < len(lens):
        while waiting and len(live) < 4:
            live.append(waiting.pop(0))
        entries, ends = [], []
        for k in live:
            if len(live) > 1 and (step + ord(k)) % 5 == 0:
                continue                # left out of this step
            n = portions[(step + ord(k)) % 7]
            toks = seqs[k][0][at[k]:at[k] + n]
            entries.append((k, toks))
            at[k] += len(toks)
            if at[k] == lens[k]:
                ends.append(k)
        out = s.step([feed(s, k, t) for k, t in entries], ends)
        row = 0
        for k, t in entries:
            got[k].append(out[row:row + len(t)])
            row += len(t)
        done |= set(ends)
        live = [k for k in live if k not in done]
        step += 1
    for k in lens:
        check(torch.cat(got[k]), seqs[k][1], where)
    cache = s.runner.cache
    assert cache.free_slots == 4 and cache.free_pages == cache.num_pages - 1


@pytest.mark.parametrize("where", WHERE)
def test_far_key_behind_the_window(model, where):
    """Changing a token that every window has passed, with no recurrence to
    remember it, must not change a logit; one inside must."""
    cfg = cases.config([latent(window=8)], taps=2)
    w = cases.weights(cfg, seed=3)
    folder = cases.save(os.path.join(model("mix")[0], "far"), cfg, w)
    toks = prompt(60)
    other = list(toks)
    other[40] = (toks[40] + 1) % 101
    s = session(folder, where, 128)
    rows = []
    for rid, t in (("a", toks), ("b", other)):
        rows.append(torch.cat(
            [s.step([feed(s, rid, t[:43])], [])] +
            [s.step([feed(s, rid, [x])], []) for x in t[43:]]))
    diff = (rows[0] - rows[1]).abs().amax(-1)
    # the convolution (two taps) reaches one token further than the window
    assert diff[:40].max() < 1e-6 and diff[49:].max() < 1e-6
    assert (diff[40:48] > 1e-4).all()


@pytest.mark.parametrize("where", WHERE)
def test_wanted_rows_and_empty_steps(model, where):
    folder = model("mix")[0]
    toks, want = want_of(model, "mix", 75)
    s = session(folder, where, 80)
    out = s.step([{"id": 1, "tokens": toks[:40], "want": []}], [])
    assert out.shape == (0, 101)
    out = s.step([{"id": 1, "tokens": toks[40:], "want": [34, 0, 7]}], [])
    check(out, want[[74, 40, 47]], where)
    assert s.step([], [1]).shape[0] == 0


def test_session_rejects_bad_input(model):
    s = session(model("mix")[0], ("cpu", "float32"), 32, max_requests=1)
    with pytest.raises(ValueError):
        s.step([{"id": 1, "tokens": [101]}], [])
    with pytest.raises(ValueError):
        s.step([{"id": 1, "tokens": [1], "want": [1]}], [])
    s.step([feed(s, 1, [1, 2])], [])
    with pytest.raises(OutOfPages):     # slots
        s.step([feed(s, 2, [1, 2])], [])
    with pytest.raises(OutOfPages):     # pages
        s.step([feed(s, 1, [1] * 40)], [])


# -- generation through the engine -------------------------------------------------


def engine(folder, where, **kw):
    cfg = load_config(folder)
    cfg.dtype = where[1]
    kw.setdefault("enforce_eager", where[0] == "cpu")
    return LLMEngine(EngineConfig(model=cfg, device=where[0],
                                  max_seq_len=128, **kw))


@pytest.mark.parametrize("where", WHERE[:2])
@pytest.mark.parametrize("mixed", [True, False])
def test_greedy_generation(model, where, mixed):
    """Prompts longer than the step's budget, more requests than slots and
    pages: the scheduler's choices must not show in the tokens."""
    folder, cfg, w = model("mix")
    prompts = [prompt(n, seed=50 + n) for n in (30, 3, 17, 1, 40)]
    eng = engine(folder, where, kv_pool_tokens=176, state_slots=3,
                 max_batch_size=4, max_prefill_tokens=16, mixed_steps=mixed)
    seqs = eng.generate(prompts, SamplingParams(max_new_tokens=12))
    for p, s in zip(prompts, seqs):
        assert len(s.output_tokens) == 12
        logits = answers(p + s.output_tokens[:-1], cfg, w)[len(p) - 1:]
        best = logits.max(-1).values
        got = logits[range(12), s.output_tokens]
        assert (best - got).max() < 1e-4        # greedy, up to a near tie
    assert eng.runner.cache.free_slots == 3
    modes = eng.stats.snapshot()
    assert modes["prefill_steps"] > 2 and modes["decode_steps"] > 0


@pytest.mark.gpu
@pytest.mark.parametrize("n", [1, 3, 5])
def test_decode_graph_replays_match_eager(model, n):
    """Captured decode steps, padded batches included, replayed many times
    with eager work between them."""
    folder = model("mix")[0]
    prompts = [prompt(5 + 9 * i, seed=70 + i) for i in range(n)]
    outs = []
    for eager in (True, False):
        eng = engine(folder, ("cuda", "bfloat16"), kv_pool_tokens=2048,
                     max_batch_size=8, enforce_eager=eager)
        seqs = [eng.add_request(p, SamplingParams(max_new_tokens=20))
                for p in prompts]
        logits = []
        runner = eng.runner
        inner = runner._decode_logits

        def keep(s):
            out = inner(s)
            logits.append(out.float().cpu())
            torch.cuda.synchronize()
            return out
        runner._decode_logits = keep
        while eng.scheduler.has_work():
            eng.step()
        outs.append((logits, [s.output_tokens for s in seqs]))
        assert bool(runner._graphs) != eager
    (a, ta), (b, tb) = outs
    assert len(a) == len(b) == 19
    steps = next((i for i, (x, y) in enumerate(zip(zip(*ta), zip(*tb)))
                  if x != y), 20)
    assert steps > 5                    # a near tie may part the two later on
    for x, y in list(zip(a, b))[:steps]:
        assert rel_err(x, y.double()) < 2e-2


def test_mixed_steps_are_the_models_choice():
    eng = LLMEngine(EngineConfig(model=resolve_model("tiny-bitatar"),
                                 device="cpu", kv_pool_tokens=256))
    assert eng.scheduler.mixed_steps and eng.runner.cache.prefix is None
    with pytest.raises(ValueError):
        LLMEngine(EngineConfig(model=resolve_model("tiny"), device="cpu",
                               kv_pool_tokens=256, mixed_steps=True))


def test_reload_weights(model):
    folder = model("mix")[0]
    eng = engine(folder, ("cpu", "float32"), kv_pool_tokens=256)
    p = [prompt(9)]
    (a,) = eng.generate(p, SamplingParams(max_new_tokens=4))
    with torch.no_grad():
        eng.runner.model.lm_head.zero_()
    eng.reload_weights(seed=1)          # a model with a file reads it again
    (b,) = eng.generate(p, SamplingParams(max_new_tokens=4))
    assert a.output_tokens == b.output_tokens
    rnd = LLMEngine(EngineConfig(model=resolve_model("tiny-bitatar"),
                                 device="cpu", kv_pool_tokens=256))
    (a,) = rnd.generate(p, SamplingParams(max_new_tokens=4))
    rnd.reload_weights(seed=99)
    (b,) = rnd.generate(p, SamplingParams(max_new_tokens=4))
    assert a.output_tokens != b.output_tokens


# -- cache, migration, loader, command line --------------------------------------


def test_migration_carries_pages_and_state(model):
    """A sequence prefilled in one engine goes on in another's pages and slot
    from the exported bytes."""
    folder, cfg, w = model("mix")
    toks, want = want_of(model, "mix", 75)
    src = session(folder, ("cpu", "float32"), 80)
    dst = session(folder, ("cpu", "float32"), 160)
    dst.step([feed(dst, "other", toks[:20])], [])     # shift pages and slots
    src.step([feed(src, "a", toks[:50])], [])
    seq = src.live["a"]
    cache, peer = src.runner.cache, dst.runner.cache
    buf = cache.export_pages(seq.block_table.pages, seq.block_table.state_slot)
    shape, dtype = peer.export_shape(len(seq.block_table.pages))
    assert tuple(buf.shape) == tuple(shape) and buf.dtype == dtype
    table = BlockTable(peer)
    table.pages = peer.alloc(len(seq.block_table.pages))
    peer.import_pages(table.pages, buf, table.state_slot)
    assert table.pages != seq.block_table.pages
    seq.block_table, dst.live["a"] = table, seq
    out = dst.step([feed(dst, "a", toks[50:])], [])
    check(out, want[50:], ("cpu", "float32"))


def test_loader_checks_names_shapes_and_config(model, tmp_path):
    _, cfg, w = model("odd")

    def load(c, ws, sub):
        m = load_config(cases.save(tmp_path / sub, c, ws))
        m.dtype = "float32"
        return TraceSession(m, 16, device="cpu")
    load(cfg, w, "ok")
    # a norm whose branch the layer does not have may be in the file
    load(cfg, dict(w, **{"l1.norm2": torch.ones(35).bfloat16()}), "spare")
    with pytest.raises(ValueError, match="does not use|do not use|not use"):
        load(cfg, dict(w, extra=torch.ones(3)), "extra")
    with pytest.raises(KeyError, match="l1.mix.w2"):
        load(cfg, {n: t for n, t in w.items() if n != "l1.mix.w2"}, "miss")
    with pytest.raises(ValueError, match="head"):
        load(cfg, dict(w, head=torch.ones(3, 3)), "shape")
    bad = json.loads(json.dumps(cfg))
    bad["layers"][0]["type"] = "other"
    with pytest.raises(ValueError, match="other"):
        load(bad, w, "type")
    bad = dict(cfg, architecture="Nobody")
    with pytest.raises(ValueError, match="Nobody"):
        load(bad, w, "arch")


@pytest.mark.parametrize("where", WHERE)
def test_trace_run(model, where, tmp_path):
    folder = model("mix")[0]
    toks, want = want_of(model, "mix", 75)
    steps = [
        {"step": 0, "entries": [feed(None, "a", toks[:60]),
                                feed(None, "b", toks[:1], want=False)],
         "end": []},
        {"step": 1, "entries": [feed(None, "b", toks[1:4], want=False),
                                feed(None, "a", [toks[60]])], "end": ["a"]},
        {"step": 2, "entries": [{"id": "b", "tokens": toks[4:9],
                                 "want": [4, 1]}], "end": ["b"]},
        {"step": 3, "entries": [feed(None, "b", toks[:5], want=False)],
         "end": ["b"]}]
    res = subprocess.run(
        [os.path.join(ROOT, "bin", "trace_run"), "--model", folder, "--dtype",
         where[1], "--out", str(tmp_path), "--max-tokens", "128",
         "--device", where[0]],
        input="".join(json.dumps(s) + "\n" for s in steps), text=True,
        capture_output=True, timeout=280, cwd=str(tmp_path))
    assert res.returncode == 0, res.stderr[-2000:]
    assert [ln for ln in res.stdout.splitlines() if ln.startswith("done")] == \
        [f"done {i}" for i in range(4)]
    assert sorted(f for f in os.listdir(tmp_path) if f.endswith(".f32")) == \
        ["0.f32", "1.f32", "2.f32"]

    def read(i):
        raw = (tmp_path / f"{i}.f32").read_bytes()
        return torch.frombuffer(bytearray(raw), dtype=torch.float32).view(
            -1, 101)
    check(read(0), want[:60], where)
    check(read(1), want[60:61], where)
    check(read(2), want[[8, 5]], where)


def test_trace_run_refuses_an_unknown_dtype(model):
    res = subprocess.run(
        [sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model",
         model("mix")[0], "--dtype", "float8", "--out", ".", "--max-tokens",
         "64"], input="", text=True, capture_output=True, timeout=60)
    assert res.returncode != 0
