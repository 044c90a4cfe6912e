"""Danipel through the framework — loader, cache, batches, scheduler, generation,
command line — against the plain oracle.  On the CPU the reference path runs; the
GPU runs (marked) take the HIP kernels, in f32 and bf16."""
import json
import os
import subprocess

import pytest
import torch

from rbg_amd.engine.config import EngineConfig
from rbg_amd.engine.engine import LLMEngine
from rbg_amd.engine.kv_cache import BlockTable, OutOfPages
from rbg_amd.engine.sequence import SamplingParams
from rbg_amd.models.registry import load_config, resolve_model
from tests import danipel_cases as cases
from tests.danipel_cases import (answers, dense, direct, indirect, moe, prompt,
                                 rel_err)
from tests.test_gogalix import WHERE, check, engine, feed, session

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))

MODELS = {
    # every branch: both attentions, both feed-forwards and none, with and
    # without scaled rotation, identity and shared experts; unequal sizes
    "mix": cases.config([
        direct(), indirect(mlp=moe()),
        direct(heads=2, dim=24, rot_dim=16, vdim=8, kv_rank=24, scale=0.2,
               scaling=None, base=5e4, mlp=moe(identity=0, shared=None)),
        indirect(heads=5, dim=8, rot_dim=16, vdim=16, kv_rank=64, q_rank=24,
                 mlp=None),
        direct(kv_rank=16, mlp=moe(ff=40, n=2, identity=2, top=3, scale=0.7,
                                   limit=3.0, shared=(8, 2.0)))], streams=3),
    # sizes that no vector access divides, one head, one stream, every expert
    # chosen
    "odd": cases.config([
        direct(heads=1, dim=5, rot_dim=2, vdim=7, kv_rank=11, mlp=dense(21)),
        indirect(heads=3, dim=3, rot_dim=6, vdim=5, kv_rank=9, q_rank=13,
                 scaling=cases.YARN,
                 mlp=moe(ff=13, n=1, identity=2, top=3, shared=(7, 0.8))),
        direct(heads=2, dim=7, rot_dim=10, vdim=3, kv_rank=6, mlp=None)],
        width=35, vocab=67, eps=1e-2, scale=1.0, streams=1, mult=1.0),
    # sizes of whole tiles, many streams
    "wide": cases.config([
        direct(heads=16, dim=32, rot_dim=32, vdim=64, kv_rank=96, scale=0.12),
        indirect(heads=17, dim=64, rot_dim=64, vdim=64, kv_rank=256,
                 q_rank=64, scale=0.09,
                 mlp=moe(ff=32, n=8, identity=4, top=3))],
        width=64, streams=4, mult=0.4),
    "five": cases.config([direct(), indirect()], streams=5, mult=0.3),
}
# weights whose routers leave a margin between chosen and left out
SEEDS = {"mix": 1, "wide": 2}


@pytest.fixture(scope="module")
def model(tmp_path_factory):
    """name -> (folder, config, weights)"""
    made = {}

    def get(name):
        if name not in made:
            cfg = MODELS[name]
            w = cases.weights(cfg, seed=SEEDS.get(name, 0))
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


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("name", MODELS)
def test_whole_prompt_then_token_by_token(model, where, name):
    """One portion; the same token by token from an empty sequence; and a
    long decode after a short portion."""
    folder = model(name)[0]
    toks, want = want_of(model, name, 75)
    s = session(folder, where, 80)
    check(s.step([feed("a", toks)], ["a"]), want, where)
    # the freed pages serve the next request
    rows = [s.step([feed("b", [t])], []) for t in toks]
    check(torch.cat(rows), want, where)
    s.step([], ["b"])
    rows = [s.step([feed("c", toks[:3])], [])]
    rows += [s.step([feed("c", [t])], []) for t in toks[3:]]
    check(torch.cat(rows), want, where)


@pytest.mark.parametrize("where", WHERE)
@pytest.mark.parametrize("name,sizes", [
    ("mix", [2]), ("mix", [3, 16, 1, 2, 33]), ("odd", [2, 5]),
    ("wide", [17, 2, 15, 1]), ("five", [2, 9, 1])])
def test_portions(model, where, name, sizes):
    """Cut anywhere, also inside pages, down to two tokens."""
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
def test_mixed_batches_reuse_pages(model, where, name):
    """Unequal requests in every phase together, with barely enough pages; each
    pauses now and then and goes on."""
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
    assert cache.free_pages == cache.num_pages - 1


@pytest.mark.parametrize("where", WHERE)
def test_long_decode(model, where):
    """Two hundred decoded tokens after a short prompt, past the length that
    the rotation was scaled from."""
    folder = model("wide")[0]
    toks, want = want_of(model, "wide", 210, seed=5)
    s = session(folder, where, 224)
    rows = [s.step([feed(0, toks[:9])], [])]
    rows += [s.step([feed(0, [t])], []) for t in toks[9:]]
    check(torch.cat(rows), want, where)


@pytest.mark.parametrize("where", WHERE[:2])
@pytest.mark.parametrize("kind", [direct, indirect])
@pytest.mark.parametrize("at", [0, 15, 16, 47])
def test_a_far_token_shows(model, where, kind, at):
    """A changed token, the first or one beside a page's border, changes every
    later row and none before it, in prompts and decoded alone."""
    cfg = cases.config([kind(rot_dim=16, mlp=None)], streams=2)
    w = cases.weights(cfg, seed=3, sharpen=0.3)
    folder = cases.save(os.path.join(model("five")[0], kind.__name__), cfg, w)
    toks = prompt(150, seed=4)
    other = list(toks)
    other[at] = (toks[at] + 1) % cases.VOCAB
    s = session(folder, where, 320)
    rows = []
    for rid, t in (("a", toks), ("b", other)):
        rows.append(torch.cat(
            [s.step([feed(rid, t[:101])], [])] +
            [s.step([feed(rid, [x])], []) for x in t[101:]]))
    diff = (rows[0] - rows[1]).abs().amax(-1)
    assert not at or diff[:at].max() < 1e-6
    assert (diff[at:] > 1e-5).all()


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


def test_pages_run_out(model):
    s = session(model("mix")[0], ("cpu", "float32"), 32, max_requests=1)
    s.step([feed(1, [1, 2])], [])
    with pytest.raises(OutOfPages):
        s.step([feed(1, [1] * 40)], [])


# -- generation through the engine -------------------------------------------------


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
    """Prompts longer than the step's budget, more requests than pages: the
    scheduler's choices must not show in the tokens."""
    folder, cfg, w = model("mix")
    prompts = [prompt(n, seed=50 + n) for n in (30, 3, 17, 1, 40)]
    eng = engine(folder, where, kv_pool_tokens=176, max_batch_size=4,
                 max_prefill_tokens=16, mixed_steps=mixed)
    seqs = eng.generate(prompts, SamplingParams(max_new_tokens=12))
    assert_greedy(prompts, seqs, cfg, w, 12)
    modes = eng.stats.snapshot()
    assert modes["prefill_steps"] > 2 and modes["decode_steps"] > 0


@pytest.mark.parametrize("where", WHERE[:2])
def test_prefix_reuse(model, where):
    """Pages are all a sequence has: prompts with a common beginning share
    them, rotated key parts included."""
    folder, cfg, w = model("five")
    head = prompt(37, seed=9)
    prompts = [head + prompt(n, seed=n) for n in (5, 1, 20)] + [head[:33]]
    eng = engine(folder, where, kv_pool_tokens=1024)
    seqs = []
    for p in prompts:
        seqs += eng.generate([p], SamplingParams(max_new_tokens=6))
    assert eng.runner.cache.prefix.hits >= 6
    assert_greedy(prompts, seqs, cfg, w, 6)


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
    rnd = LLMEngine(EngineConfig(model=resolve_model("tiny-danipel"),
                                 device="cpu", kv_pool_tokens=256,
                                 max_seq_len=256, max_batch_size=4))
    assert rnd.scheduler.mixed_steps
    (a,) = rnd.generate(p, SamplingParams(max_new_tokens=4))
    rnd.reload_weights(seed=99)
    (b,) = rnd.generate(p, SamplingParams(max_new_tokens=4))
    assert a.output_tokens != b.output_tokens


# -- cache, migration, loader, command line --------------------------------------


def test_cache_holds_latents_and_rotated_parts(model):
    cfg = MODELS["mix"]
    cache = session(model("mix")[0], ("cpu", "float32"), 64).runner.cache
    per_token = sum(la["mixer"]["kv_rank"] + la["mixer"]["rot_dim"]
                    for la in cfg["layers"])
    assert cache.kv.numel() == per_token * cache.num_pages * 16
    assert cache.latents(3).shape[1:] == (16, 64 + 16)
    assert not cache.has_state


def test_migration_carries_pages(model):
    """A sequence prefilled in one engine goes on in another's pages from the
    exported bytes."""
    folder = model("mix")[0]
    toks, want = want_of(model, "mix", 75)
    src = session(folder, ("cpu", "float32"), 80)
    dst = session(folder, ("cpu", "float32"), 160)
    dst.step([feed("other", toks[:20])], [])     # shift pages
    src.step([feed("a", toks[:50])], [])
    seq = src.live["a"]
    cache, peer = src.runner.cache, dst.runner.cache
    buf = cache.export_pages(seq.block_table.pages)
    shape, dtype = peer.export_shape(len(seq.block_table.pages))
    assert tuple(buf.shape) == tuple(shape) and buf.dtype == dtype
    table = BlockTable(peer)
    table.pages = peer.alloc(len(seq.block_table.pages))
    peer.import_pages(table.pages, buf)
    assert table.pages != seq.block_table.pages
    seq.block_table, dst.live["a"] = table, seq
    out = dst.step([feed("a", toks[50:])], [])
    check(out, want[50:], ("cpu", "float32"))


def test_loader_checks_names_shapes_and_config(model, tmp_path):
    _, cfg, w = model("mix")

    def load(c, ws, sub):
        m = load_config(cases.save(tmp_path / sub, c, ws))
        m.dtype = "float32"
        return session(str(tmp_path / sub), ("cpu", "float32"), 16)
    load(cfg, w, "ok")
    # what a feed-forward would need may be in the file without one
    load(cfg, dict(w, **{"l3.hc2.in": torch.ones(3).bfloat16()}), "spare")
    with pytest.raises(ValueError, match="not use"):
        load(cfg, dict(w, **{"l1.mix.sink": torch.ones(3)}), "extra")
    with pytest.raises(KeyError, match="l1.mlp.e3.down"):
        load(cfg, {n: t for n, t in w.items() if n != "l1.mlp.e3.down"},
             "miss")
    with pytest.raises(KeyError, match="l0.mix.sink"):
        load(cfg, {n: t for n, t in w.items() if n != "l0.mix.sink"}, "sink")
    with pytest.raises(ValueError, match="l0.norm1.alpha"):
        load(cfg, dict(w, **{"l0.norm1.alpha": torch.ones(48)}), "shape")

    def broken(change, match):
        bad = json.loads(json.dumps(cfg))
        change(bad)
        with pytest.raises(ValueError, match=match):
            load(bad, w, "bad")
    broken(lambda c: c["layers"][0].update(type="other"), "other")
    broken(lambda c: c["layers"][0].update(mlp={"kind": "wide"}), "wide")
    broken(lambda c: c["layers"][0]["mixer"]["rot"].update(dims=6), "6 rotated")
    broken(lambda c: c["layers"][0]["mixer"].update(heads=4), "l0.mix.q")
    broken(lambda c: c["layers"][1]["mlp"]["router"].update(top=9), "chosen")
    broken(lambda c: c["layers"][1]["mlp"]["router"].update(identity=2),
           "router")
    broken(lambda c: c.update(streams=0), "streams")
    broken(lambda c: c.update(streams=2), "l0.hc1")


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
        capture_output=True, timeout=110, cwd=str(tmp_path))
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
