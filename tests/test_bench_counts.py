"""bench.py counts the tokens that were decoded: every decode point's schedule is replayed
on the CPU through the real engine loop, scheduler and cache manager (the model's step is
replaced by one that returns zero logits), at the sizes bench.py uses, and `decode_run`
itself checks that every request is live through the timed steps and that the tokens it
reports are the tokens the requests received."""

import sys
from pathlib import Path

import pytest
import torch

sys.path.insert(0, str(Path(__file__).resolve().parent.parent))

import bench  # noqa: E402
from helpers import TINY_A  # noqa: E402
from kernel_refs import TorchOps  # noqa: E402
from tokensprint_amd.config import Config  # noqa: E402
from tokensprint_amd.engine.assemble import random_model  # noqa: E402
from tokensprint_amd.engine.llm_engine import LLMEngine  # noqa: E402


@pytest.fixture(scope="module")
def model():
    cfg = dict(TINY_A, max_position_embeddings=8192)
    return random_model(cfg, 0, "float32", "cpu", ops=TorchOps())[1]


def fake_engine(model, tmp_path, batch, max_len, budget, page=16):
    engine = LLMEngine(model, Config(
        model=str(tmp_path), max_model_len=max_len, dtype=torch.float32,
        kvcache_block_size=page, num_kvcache_blocks=batch * (-(-max_len // page) + 1),
        max_num_seqs=batch, max_num_batched_tokens=budget, chunked_prefill=True, eos=-1))
    vocab = model.spec.vocab_size
    engine.runner.step = lambda entries: torch.zeros(
        sum(len(e.want) for e in entries), vocab)
    return engine


@pytest.mark.parametrize("steps,warmup", [(20, 5), (496, 16)])
def test_every_point_counts_what_it_decodes(model, tmp_path, steps, warmup):
    plan = bench.decode_points(8, 512, steps, warmup)
    assert list(plan)[0] == "headline" and {"decode_b1", "decode_b64"} <= set(plan)
    for name, (b, prompt_len, k, w, budget) in plan.items():
        max_len, max_tokens = bench.decode_lengths(b, prompt_len, k, w, budget)
        engine = fake_engine(model, tmp_path, b, max_len, budget)
        _, decoded, held = bench.decode_run(engine, b, prompt_len, k, w, 256, max_tokens)
        assert decoded == b * k, name
        # every request held its prompt and at least the warm-up's tokens all along
        assert held / b >= prompt_len + w + k / 2, name
        assert all(pool.num_used == 0 for pool in engine.runner.manager.pools), name


def test_a_request_that_leaves_early_is_an_error(model, tmp_path):
    engine = fake_engine(model, tmp_path, 64, 1024, 2048)
    with pytest.raises(RuntimeError, match="live before"):
        # room for fewer tokens than the prompts' skew and the steps need
        bench.decode_run(engine, 64, 512, 20, 5, 256, max_tokens=30)


def test_compared_designs_are_of_equal_size():
    """`bench.py --compare-zonopel` builds a Zonopel and a Qwen3 configuration per size with
    the same width, depth, vocabulary and (within 2 %) number of parameters."""
    import math

    import bench
    from tokensprint_amd.weights.random_init import declared_tensors
    for name, size in bench.COMPARE_SIZES.items():
        zono, qwen = bench.compare_configs(size)
        count = [sum(math.prod(d.shape) for d in declared_tensors(raw).values())
                 for raw in (zono, qwen)]
        assert abs(count[0] - count[1]) <= 0.02 * count[0], (name, count)
        assert zono["width"] == qwen["hidden_size"] and zono["vocab"] == qwen["vocab_size"]
        assert len(zono["layers"]) == qwen["num_hidden_layers"]
        assert {e["type"] for e in zono["layers"]} == {"mamba2", "latent_attention"}


def test_palelix_and_zonopel_are_compared_at_equal_size():
    """`bench.py --compare-palelix` builds a Palelix and a Zonopel configuration per size with
    the same width, depth, vocabulary and (within 2 %) number of parameters, every kind of
    mixer and both kinds of feed-forward among the Palelix layers."""
    import math

    import bench
    from tokensprint_amd.weights.random_init import declared_tensors
    for name, size in bench.COMPARE_SIZES.items():
        pale, zono = bench.palelix_configs(size)
        count = [sum(math.prod(d.shape) for d in declared_tensors(raw).values())
                 for raw in (pale, zono)]
        assert abs(count[0] - count[1]) <= 0.02 * count[0], (name, count)
        assert pale["width"] == zono["width"] and pale["vocab"] == zono["vocab"]
        assert len(pale["layers"]) == len(zono["layers"])
        assert {e["type"] for e in pale["layers"]} == {"delta", "lightning", "parallel"}
        assert {e["mlp"]["kind"] for e in pale["layers"]} == {"dense", "moe"}


def test_zolorax_and_zonopel_are_compared_at_equal_size():
    """`bench.py --compare-zolorax` builds a Zolorax and a Zonopel configuration per size with
    the same width, depth, vocabulary and (within 2 %) number of parameters, both kinds of
    mixer, a layer that reads another's keys, and both kinds of feed-forward."""
    import math

    import bench
    from tokensprint_amd.weights.random_init import declared_tensors
    for name, size in bench.COMPARE_SIZES.items():
        zolo, zono = bench.zolorax_configs(size)
        count = [sum(math.prod(d.shape) for d in declared_tensors(raw).values())
                 for raw in (zolo, zono)]
        assert abs(count[0] - count[1]) <= 0.02 * count[0], (name, count)
        assert zolo["width"] == zono["width"] and zolo["vocab"] == zono["vocab"]
        assert len(zolo["layers"]) == len(zono["layers"])
        assert {e["type"] for e in zolo["layers"]} == {"rglru", "attention"}
        assert any("kv_from" in e["mixer"] for e in zolo["layers"])
        assert {e["mlp"]["kind"] for e in zolo["layers"]} == {"dense", "moe"}


def test_fubepel_and_zonopel_are_compared_at_equal_size():
    """`bench.py --compare-fubepel` builds a Fubepel and a Zonopel configuration per size with
    the same width, depth, vocabulary and (within 2 %) number of parameters, every kind of
    mixer and a layer that reads another's latents."""
    import math

    import bench
    from tokensprint_amd.weights.random_init import declared_tensors
    for name, size in bench.COMPARE_SIZES.items():
        fube, zono = bench.fubepel_configs(size)
        count = [sum(math.prod(d.shape) for d in declared_tensors(raw).values())
                 for raw in (fube, zono)]
        assert abs(count[0] - count[1]) <= 0.02 * count[0], (name, count)
        assert fube["width"] == zono["width"] and fube["vocab"] == zono["vocab"]
        assert len(fube["layers"]) == len(zono["layers"])
        assert {e["type"] for e in fube["layers"]} == {"latent_attention", "delta", "attention"}
        assert any("kv_from" in e["mixer"] for e in fube["layers"]) and fube["token_side"]


def test_sisepel_and_palelix_are_compared_at_equal_size():
    """`bench.py --compare-sisepel` builds a Sisepel and a Palelix configuration per size with
    the same width, depth, vocabulary and (within 2 %) number of parameters, every option and
    both kinds of feed-forward, and retention of the size of the other's linear attention."""
    import math

    import bench
    from tokensprint_amd.weights.random_init import declared_tensors
    for name, size in bench.COMPARE_SIZES.items():
        sise, pale = bench.sisepel_configs(size)
        count = [sum(math.prod(d.shape) for d in declared_tensors(raw).values())
                 for raw in (sise, pale)]
        assert abs(count[0] - count[1]) <= 0.02 * count[0], (name, count)
        assert sise["width"] == pale["width"] and sise["vocab"] == pale["vocab"]
        assert len(sise["layers"]) == len(pale["layers"])
        assert {e["mlp"]["kind"] for e in sise["layers"]} == {"dense", "moe"}
        left, right = (sise["layers"][1]["mixer"][side] for side in ("left", "right"))
        assert {"softcap", "mask", "rot"} <= set(left) and sise["token_side"]
        other = next(e["mixer"] for e in pale["layers"] if e["type"] == "lightning")
        assert [right[k] for k in ("heads", "dim", "vdim")] == [other[k] for k in ("heads", "dim", "vdim")]
