"""Bitatar served by the framework's roles on the CPU (tiny preset): colocated,
prefill/decode with state migration, and sharded over two ranks (gloo)."""
import pytest
import torch

from rbg_amd.api.types import ObjectMeta, RoleBasedGroup, RoleBasedGroupSpec
from tests import bitatar_cases as cases
from tests.test_controller_e2e import rbg_ready
from tests.test_parallel import _free_port, _init, _run_dist
from tests.test_serving_e2e import (_http_post, _router_http_port,  # noqa: F401
                                    engine_role, mgr, router_role)


def local_tokens(model, prompt, max_new):
    from rbg_amd.engine.config import EngineConfig
    from rbg_amd.engine.engine import LLMEngine
    from rbg_amd.engine.sequence import SamplingParams
    from rbg_amd.models.registry import resolve_model
    eng = LLMEngine(EngineConfig(model=resolve_model(model), device="cpu",
                                 kv_pool_tokens=1024, state_slots=4,
                                 enforce_eager=True))
    (s,) = eng.generate([prompt], SamplingParams(max_new_tokens=max_new))
    return s.output_tokens


def serve(mgr, name, roles):  # noqa: F811
    mgr.store.create(RoleBasedGroup(metadata=ObjectMeta(name=name),
                                    spec=RoleBasedGroupSpec(roles=roles)))
    assert mgr.wait_for(lambda: rbg_ready(mgr, name), timeout=180)
    assert mgr.wait_for(lambda: _router_http_port(mgr, name) is not None,
                        timeout=30)
    return _router_http_port(mgr, name)


@pytest.mark.timeout(300)
def test_colocated_from_a_model_folder(mgr, tmp_path):  # noqa: F811
    cfg = cases.config([cases.delta(), cases.latent(window=9)])
    folder = cases.save(tmp_path / "m", cfg, cases.weights(cfg))
    port = serve(mgr, "bit", [
        router_role("colocated", {"worker_roles": ["worker"],
                                  "vocab_size": 101}),
        engine_role("worker", "colocated", {"model": folder})])
    for n in (12, 33):
        prompt = cases.prompt(n, seed=n)
        res = _http_post(port, "/generate", {"prompt_tokens": prompt,
                                             "max_new_tokens": 6})
        assert res["tokens"] == local_tokens(folder, prompt, 6)


@pytest.mark.timeout(300)
def test_prefill_decode_roles_migrate_state(mgr):  # noqa: F811
    shared = {"comm_backend": "gloo", "model": "tiny-bitatar",
              "prefill_roles": ["prefill"], "decode_roles": ["decode"],
              # fewer slots than requests: a parked prefill holds one
              "state_slots": 2}
    port = serve(mgr, "bitpd", [
        router_role("pd", {"prefill_roles": ["prefill"],
                           "decode_roles": ["decode"], "vocab_size": 500}),
        engine_role("prefill", "prefill", shared),
        engine_role("decode", "decode", shared)])
    for n in (25, 9, 40):
        prompt = cases.prompt(n, vocab=500, seed=n)
        res = _http_post(port, "/generate", {"prompt_tokens": prompt,
                                             "max_new_tokens": 6})
        assert res["tokens"] == local_tokens("tiny-bitatar", prompt, 6)


def _shard_worker(rank, world, port, kind, folder, prompts, path):
    torch.set_num_threads(1)
    dist = _init(rank, world, port)
    from rbg_amd.engine.config import EngineConfig
    from rbg_amd.engine.engine import LLMEngine
    from rbg_amd.engine.sequence import SamplingParams
    from rbg_amd.models.llama import PPContext, TPContext
    from rbg_amd.models.registry import load_config
    cfg = load_config(folder)
    cfg.dtype = "float32"
    tp = pp = None
    if kind == "tp":
        tp = TPContext(size=world, rank=rank)
    else:
        pp = PPContext(size=world, stage=rank, instance_ranks=[0, 1])
    eng = LLMEngine(EngineConfig(model=cfg, device="cpu", kv_pool_tokens=512,
                                 state_slots=3, max_prefill_tokens=16,
                                 tp_size=world if tp else 1, tp_rank=rank),
                    tp, pp)
    seqs = eng.generate(prompts, SamplingParams(max_new_tokens=8))
    if rank == world - 1:
        torch.save([s.output_tokens for s in seqs], path)
    dist.barrier()
    dist.destroy_process_group()


@pytest.mark.parametrize("kind", ["tp", "pp"])
def test_two_ranks_match_one(kind, tmp_path):
    cfg = cases.config([cases.delta(heads=4), cases.latent(heads=2),
                        cases.latent(heads=4, window=6, ff=None),
                        cases.delta(heads=2)])
    folder = cases.save(tmp_path / "m", cfg, cases.weights(cfg, seed=8))
    prompts = [cases.prompt(n, seed=n) for n in (20, 3, 11)]
    _run_dist(_shard_worker, 2, _free_port(), kind, folder, prompts,
              str(tmp_path / "out.pt"))
    from rbg_amd.engine.config import EngineConfig
    from rbg_amd.engine.engine import LLMEngine
    from rbg_amd.engine.sequence import SamplingParams
    from rbg_amd.models.registry import load_config
    one = load_config(folder)
    one.dtype = "float32"
    eng = LLMEngine(EngineConfig(model=one, device="cpu", kv_pool_tokens=512))
    seqs = eng.generate(prompts, SamplingParams(max_new_tokens=8))
    assert torch.load(str(tmp_path / "out.pt")) == \
        [s.output_tokens for s in seqs]
