"""Danipel served by the framework's roles on the CPU: colocated from a model
folder, prefill/decode with migration of pages, and sharded over two ranks
(gloo)."""
import pytest
import torch

from tests import danipel_cases as cases
from tests.test_bitatar_serving import (_shard_worker, local_tokens, mgr,  # noqa: F401,E501
                                        serve)
from tests.test_parallel import _free_port, _run_dist
from tests.test_serving_e2e import _http_post, engine_role, router_role


@pytest.mark.timeout(300)
def test_colocated_from_a_model_folder(mgr, tmp_path):  # noqa: F811
    cfg = cases.config([cases.direct(), cases.indirect(mlp=cases.moe())])
    folder = cases.save(tmp_path / "m", cfg, cases.weights(cfg))
    port = serve(mgr, "dan", [
        router_role("colocated", {"worker_roles": ["worker"],
                                  "vocab_size": 101}),
        engine_role("worker", "colocated", {"model": folder})])
    for n in (12, 33):
        tokens = cases.prompt(n, seed=n)
        res = _http_post(port, "/generate", {"prompt_tokens": tokens,
                                             "max_new_tokens": 6})
        assert res["tokens"] == local_tokens(folder, tokens, 6)


@pytest.mark.timeout(300)
def test_prefill_decode_roles_migrate(mgr):  # noqa: F811
    shared = {"comm_backend": "gloo", "model": "tiny-danipel",
              "prefill_roles": ["prefill"], "decode_roles": ["decode"]}
    port = serve(mgr, "danpd", [
        router_role("pd", {"prefill_roles": ["prefill"],
                           "decode_roles": ["decode"], "vocab_size": 500}),
        engine_role("prefill", "prefill", shared),
        engine_role("decode", "decode", shared)])
    for n in (25, 9, 40):
        tokens = cases.prompt(n, vocab=500, seed=n)
        res = _http_post(port, "/generate", {"prompt_tokens": tokens,
                                             "max_new_tokens": 6})
        assert res["tokens"] == local_tokens("tiny-danipel", tokens, 6)


@pytest.mark.parametrize("kind", ["tp", "pp"])
def test_two_ranks_match_one(kind, tmp_path):
    cfg = cases.config([
        cases.direct(heads=4, mlp=cases.moe()),
        cases.indirect(heads=2, mlp=None),
        cases.indirect(heads=6, mlp=cases.moe(identity=0, shared=None)),
        cases.direct(heads=2)], streams=3)
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
