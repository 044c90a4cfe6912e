"""Gogalix through the framework — loader, cache, slots, batches, scheduler,
generation, command line — against the plain oracle.  On the CPU the reference
path runs; the GPU runs (marked) take the HIP kernels, in f32 and bf16."""
import json
import os
import subprocess

import pytest
import torch

from rbg_amd.engine.config import EngineConfig
from rbg_amd.engine.engine import LLMEngine
from rbg_amd.engine.kv_cache import BlockTable, OutOfPages
from rbg_amd.engine.sequence import SamplingParams
from rbg_amd.engine.trace import TraceSession
from rbg_amd.models.registry import load_config, resolve_model
from tests import gogalix_cases as cases
from tests.gogalix_cases import (answers, attention, channel, delta, dense,
                                 moe, prompt, rel_err, row_errs)

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
GPU = pytest.mark.gpu
WHERE = [pytest.param(("cpu", "float32"), id="cpu-f32"),
         pytest.param(("cuda", "float32"), id="gpu-f32", marks=GPU),
         pytest.param(("cuda", "bfloat16"), id="gpu-bf16", marks=GPU)]
# positions, relative to the answers' RMS: almost all of them, and the worst.
# bf16's rounding is magnified where a head's output almost cancels before its
# norm, so the worst one has room; f32 has none.
TOL = {"float32": (4e-5, 4e-5), "bfloat16": (5e-2, 0.2)}

MODELS = {
    # every branch: both rules, own and shared keys under unequal windows,
    # both feed-forwards and none, unequal sizes throughout
    "mix": cases.config([
        channel(), attention(mlp=moe()),
        attention(kv_from=1, window=30, scale=0.7, diff=0.6),
        delta(heads=6, kv_heads=2, dim=24, vdim=8, taps=4, mlp=moe(ff=40, n=4,
                                                                  top=1)),
        attention(heads=3, kv_heads=3, dim=16, vdim=16, window=5, mlp=None),
        channel(heads=2, kv_heads=1, dim=40, vdim=32, taps=2, mlp=None)]),
    # sizes that no vector access divides, windows of one token, one tap,
    # every expert chosen
    "odd": cases.config([
        attention(heads=3, kv_heads=1, dim=5, vdim=7, window=1,
                  mlp=moe(ff=13, n=3, top=3)),
        channel(heads=3, kv_heads=1, dim=9, vdim=5, taps=1, mlp=dense(21)),
        delta(heads=1, kv_heads=1, dim=11, vdim=13, taps=6, mlp=None),
        attention(heads=3, kv_heads=1, dim=5, vdim=7, window=19, kv_from=0,
                  mlp=dense(10))],
        width=35, vocab=67, eps=1e-3, scale=1.0),
    # head sizes of whole tiles, windows at page borders
    "wide": cases.config([
        delta(heads=4, kv_heads=4, dim=32, vdim=64, taps=4),
        attention(heads=8, kv_heads=1, dim=32, vdim=64, window=16),
        channel(heads=2, kv_heads=2, dim=128, vdim=128, taps=4,
                mlp=moe(ff=32, n=8, top=3)),
        attention(heads=2, kv_heads=2, dim=64, vdim=96, window=33,
                  scale=0.12)], width=64),
    # no attention at all: pages of no size; and no recurrence: no slots
    "rec": cases.config([delta(), channel(dim=8)]),
    "att": cases.config([attention(window=24), attention(kv_from=0, window=7),
                         attention(kv_from=0, window=40)]),
}
RANKS = {"odd": (3, 1), "wide": (16, 8)}
# weights whose routers leave a margin between chosen and left out
SEEDS = {"mix": 1, "odd": 2, "wide": 1}


@pytest.fixture(scope="module")
def model(tmp_path_factory):
    """name -> (folder, config, weights)"""
    made = {}

    def get(name):
        if name not in made:
            cfg = MODELS[name]
            w = cases.weights(cfg, seed=SEEDS.get(name, 0),
                              ranks=RANKS.get(name, (5, 12)))
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


def feed(rid, toks, want=True):
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
    check(s.step([feed("a", toks)], ["a"]), want, where)
    # the freed slot and pages serve the next request
    rows = [s.step([feed("b", [t])], []) for t in toks]
    check(torch.cat(rows), want, where)
    s.step([], ["b"])
    rows = [s.step([feed("c", toks[:3])], [])]
    rows += [s.step([feed("c", [t])], []) for t in toks[3:]]
    check(torch.cat(rows), want, where)


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("name,sizes", [
    ("mix", [2]), ("mix", [3, 16, 1, 2, 33]), ("odd", [2, 5]),
    ("wide", [17, 2, 15, 1]), ("rec", [2, 3]), ("att", [2, 9, 1])])
def test_portions(model, where, name, sizes):
    """Cut anywhere: inside pages, windows, chunks and the convolution's past,
    down to two tokens."""
    folder = model(name)[0]
    toks, want = want_of(model, name, 75)
    s = session(folder, where, 80)
    rows, at, i = [], 0, 0
    while at < len(toks):
        n = min(sizes[i % len(sizes)], len(toks) - at)
        rows.append(s.step([feed(0, toks[at:at + n])], []))
        at, i = at + n, i + 1
    check(torch.cat(rows), want, where)


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("name", ["mix", "odd", "wide"])
def test_mixed_batches_reuse_pages_and_slots(model, where, name):
    """Unequal requests in every phase together, with barely enough pages and
    two slots fewer than requests; each pauses now and then and goes on."""
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
        out = s.step([feed(k, t) for k, t in entries], ends)
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
def test_long_decode(model, where):
    """Two hundred decoded tokens after a short prompt: states and windows
    that have long forgotten it."""
    folder = model("wide")[0]
    toks, want = want_of(model, "wide", 210, seed=5)
    s = session(folder, where, 224)
    rows = [s.step([feed(0, toks[:9])], [])]
    rows += [s.step([feed(0, [t])], []) for t in toks[9:]]
    check(torch.cat(rows), want, where)


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("window,split", [(8, 43), (16, 33), (17, 48)])
def test_a_windows_edge(model, where, window, split):
    """Changing a token changes exactly the rows whose window holds it, in
    prompts and decoded alone."""
    cfg = cases.config([attention(window=window)])
    w = cases.weights(cfg, seed=3)
    folder = cases.save(os.path.join(model("rec")[0], f"edge{window}"), cfg, w)
    s = session(folder, where, 256)
    toks = prompt(70)
    for at in (5, 40):
        other = list(toks)
        other[at] = (toks[at] + 1) % cases.VOCAB
        rows = []
        for rid, t in (("a", toks), ("b", other)):
            rows.append(torch.cat(
                [s.step([feed(rid, t[:split])], [])] +
                [s.step([feed(rid, [x])], [rid] if i == 69 else [])
                 for i, x in enumerate(t) if i >= split]))
        diff = (rows[0] - rows[1]).abs().amax(-1)
        assert diff[:at].max() < 1e-6 and diff[at + window:].max() < 1e-6
        assert (diff[at:at + window] > 1e-4).all()


@pytest.mark.parametrize("where", WHERE)
def test_a_state_remembers_a_far_token(model, where):
    """With slow decays a changed token shows in every later row, and in none
    before it."""
    cfg = cases.config([delta(), channel(dim=8)])
    w = cases.weights(cfg, seed=4)
    for n in w:
        if n.endswith("A_log"):
            w[n] = torch.full_like(w[n], -7.0)
    folder = cases.save(os.path.join(model("rec")[0], "far"), cfg, w)
    toks = prompt(150, seed=4)
    other = list(toks)
    other[5] = (toks[5] + 1) % cases.VOCAB
    s = session(folder, where, 320)
    rows = []
    for rid, t in (("a", toks), ("b", other)):
        rows.append(torch.cat(
            [s.step([feed(rid, t[:101])], [])] +
            [s.step([feed(rid, [x])], []) for x in t[101:]]))
    diff = (rows[0] - rows[1]).abs().amax(-1)
    assert diff[:5].max() < 1e-6
    assert (diff[5:] > 1e-4).all()


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


def test_pages_and_slots_run_out(model):
    s = session(model("mix")[0], ("cpu", "float32"), 32, max_requests=1)
    s.step([feed(1, [1, 2])], [])
    with pytest.raises(OutOfPages):     # slots
        s.step([feed(2, [1, 2])], [])
    with pytest.raises(OutOfPages):     # pages
        s.step([feed(1, [1] * 40)], [])


# -- generation through the engine -------------------------------------------------


def engine(folder, where, **kw):
    cfg = load_config(folder)
    cfg.dtype = where[1]
    kw.setdefault("enforce_eager", where[0] == "cpu")
    return LLMEngine(EngineConfig(model=cfg, device=where[0],
                                  max_seq_len=128, **kw))


def assert_greedy(prompts, seqs, cfg, w, n):
    for p, s in zip(prompts, seqs):
        assert len(s.output_tokens) == n
        logits = answers(p + s.output_tokens[:-1], cfg, w)[len(p) - 1:]
        best = logits.max(-1).values
        got = logits[range(n), s.output_tokens]
        assert (best - got).max() < 1e-4        # greedy, up to a near tie


@pytest.mark.parametrize("where", WHERE[:2])
@pytest.mark.parametrize("mixed", [True, False])
def test_greedy_generation(model, where, mixed):
    """Prompts longer than the step's budget, more requests than slots and
    pages: the scheduler's choices must not show in the tokens."""
    folder, cfg, w = model("mix")
    prompts = [prompt(n, seed=50 + n) for n in (30, 3, 17, 1, 40)]
    eng = engine(folder, where, kv_pool_tokens=176, max_batch_size=4,
                 state_slots=3, max_prefill_tokens=16, mixed_steps=mixed)
    seqs = eng.generate(prompts, SamplingParams(max_new_tokens=12))
    assert_greedy(prompts, seqs, cfg, w, 12)
    modes = eng.stats.snapshot()
    assert modes["prefill_steps"] > 2 and modes["decode_steps"] > 0


@pytest.mark.parametrize("where", WHERE[:2])
def test_prefix_reuse_without_recurrence(model, where):
    """A model of attention alone keeps nothing beside its pages: prompts with
    a common beginning share them.  One with a state has no prefix cache."""
    folder, cfg, w = model("att")
    head = prompt(37, seed=9)
    prompts = [head + prompt(n, seed=n) for n in (5, 1, 20)] + [head[:33]]
    eng = engine(folder, where, kv_pool_tokens=1024)
    seqs = []
    for p in prompts:
        seqs += eng.generate([p], SamplingParams(max_new_tokens=6))
    assert eng.runner.cache.prefix.hits >= 6
    assert_greedy(prompts, seqs, cfg, w, 6)
    assert engine(model("mix")[0], where,
                  kv_pool_tokens=256).runner.cache.prefix is None


@pytest.mark.gpu
@pytest.mark.parametrize("n", [1, 3, 5])
def test_decode_graph_replays_match_eager(model, n):
    """Captured decode steps, padded batches included, replayed many times
    with eager work between them."""
    folder = model("wide")[0]
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


@pytest.mark.gpu
def test_graph_decode_is_greedy(model):
    """Captured steps in f32 follow the oracle token by token."""
    folder, cfg, w = model("odd")
    prompts = [prompt(n, 67, seed=n) for n in (6, 11, 2)]
    eng = engine(folder, ("cuda", "float32"), kv_pool_tokens=1024)
    seqs = eng.generate(prompts, SamplingParams(max_new_tokens=15))
    assert eng.runner._graphs
    assert_greedy(prompts, seqs, cfg, w, 15)


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
    rnd = LLMEngine(EngineConfig(model=resolve_model("tiny-gogalix"),
                                 device="cpu", kv_pool_tokens=256,
                                 max_seq_len=256, max_batch_size=4))
    assert rnd.scheduler.mixed_steps
    (a,) = rnd.generate(p, SamplingParams(max_new_tokens=4))
    rnd.reload_weights(seed=99)
    (b,) = rnd.generate(p, SamplingParams(max_new_tokens=4))
    assert a.output_tokens != b.output_tokens


# -- cache, migration, loader, command line --------------------------------------


def test_cache_holds_what_layers_keep(model):
    cfg = MODELS["mix"]
    cache = session(model("mix")[0], ("cpu", "float32"), 64).runner.cache
    per_token = sum(m["kv_heads"] * (2 * m["dim"] + m["vdim"])
                    for la in cfg["layers"] for m in [la["mixer"]]
                    if la["type"] == "attention" and "kv_from" not in m)
    assert cache.kv.numel() == per_token * cache.num_pages * 16
    k, v = cache.kv_pages(1)
    assert k.shape[1:] == (2, 16, 16) and v.shape[1:] == (2, 16, 24)
    assert cache.state(3, "delta").shape[1:] == (6, 24, 8)
    assert cache.state(3, "delta").dtype == torch.float32
    # q, k and v of the last four tokens
    assert cache.state(3, "conv").shape[1:] == (4, 2 * 48 + 48)
    with pytest.raises(AssertionError):
        cache.kv_pages(2)
    assert not session(model("att")[0], ("cpu", "float32"),
                       64).runner.cache.has_state


def test_migration_carries_pages_and_state(model):
    """A sequence prefilled in one engine goes on in another's pages and slot
    from the exported bytes."""
    folder = model("mix")[0]
    toks, want = want_of(model, "mix", 75)
    src = session(folder, ("cpu", "float32"), 80)
    dst = session(folder, ("cpu", "float32"), 160)
    dst.step([feed("other", toks[:20])], [])     # shift pages and slots
    src.step([feed("a", toks[:50])], [])
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
    out = dst.step([feed("a", toks[50:])], [])
    check(out, want[50:], ("cpu", "float32"))


def test_loader_checks_names_shapes_and_config(model, tmp_path):
    _, cfg, w = model("mix")

    def load(c, ws, sub):
        m = load_config(cases.save(tmp_path / sub, c, ws))
        m.dtype = "float32"
        return TraceSession(m, 16, device="cpu")
    load(cfg, w, "ok")
    # what a feed-forward would need may be in the file without one
    load(cfg, dict(w, **{"l4.ls2": torch.ones(48).bfloat16()}), "spare")
    with pytest.raises(ValueError, match="not use"):
        load(cfg, dict(w, **{"l2.mix.k": torch.ones(32, 48)}), "extra")
    with pytest.raises(KeyError, match="l1.mlp.e3.down"):
        load(cfg, {n: t for n, t in w.items() if n != "l1.mlp.e3.down"},
             "miss")
    with pytest.raises(ValueError, match="l0.norm1"):
        load(cfg, dict(w, **{"l0.norm1": torch.ones(48)}), "shape")

    def broken(change, match):
        bad = json.loads(json.dumps(cfg))
        change(bad["layers"])
        with pytest.raises(ValueError, match=match):
            load(bad, w, "bad")
    broken(lambda la: la[0].update(type="other"), "other")
    broken(lambda la: la[0].update(mlp={"kind": "wide"}), "wide")
    broken(lambda la: la[1]["mixer"].update(kv_from=1), "not before")
    broken(lambda la: la[4]["mixer"].update(kv_from=2), "cannot use")
    broken(lambda la: la[4]["mixer"].update(kv_from=1), "cannot use")
    broken(lambda la: la[4]["mixer"].update(kv_from=0), "cannot use")
    broken(lambda la: la[0]["mixer"].update(heads=5), "5 heads")
    broken(lambda la: la[1]["mixer"].update(heads=3), "3 heads")
    broken(lambda la: la[1]["mlp"]["router"].update(top=7), "chosen")


@pytest.mark.parametrize("where", WHERE)
def test_trace_run(model, where, tmp_path):
    folder = model("mix")[0]
    toks, want = want_of(model, "mix", 75)
    steps = [
        {"step": 0, "entries": [feed("a", toks[:60]),
                                feed("b", toks[:1], want=False)], "end": []},
        {"step": 1, "entries": [feed("b", toks[1:4], want=False),
                                feed("a", [toks[60]])], "end": ["a"]},
        {"step": 2, "entries": [{"id": "b", "tokens": toks[4:9],
                                 "want": [4, 1]}], "end": ["b"]}]
    res = subprocess.run(
        [os.path.join(ROOT, "bin", "trace_run"), "--model", folder, "--dtype",
         where[1], "--out", str(tmp_path), "--max-tokens", "128",
         "--device", where[0]],
        input="".join(json.dumps(s) + "\n" for s in steps), text=True,
        capture_output=True, timeout=280, cwd=str(tmp_path))
    assert res.returncode == 0, res.stderr[-2000:]
    assert [ln for ln in res.stdout.splitlines() if ln.startswith("done")] == \
        [f"done {i}" for i in range(3)]

    def read(i):
        raw = (tmp_path / f"{i}.f32").read_bytes()
        return torch.frombuffer(bytearray(raw), dtype=torch.float32).view(
            -1, 101)
    check(read(0), want[:60], where)
    check(read(1), want[60:61], where)
    check(read(2), want[[8, 5]], where)
