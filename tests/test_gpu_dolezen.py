"""The Dolezen decoder on the GPU, through the engine's runner, scheduler and trace replay, against the plain
implementation: float32 tightly, bfloat16 within what rounding allows."""

from __future__ import annotations

import pytest
import torch

from llmserve_amd import CacheConfig, GenerationConfig, SchedulerConfig
from llmserve_amd.engine import EngineCore, ModelRunner, StepEntry
from llmserve_amd.weights import load_model_folder
from tests import dolezen_cases as cases
from tests.gpu_helpers import TraceBuilder, replay
from tests.plain import dolezen_plain as plain
from tests.test_dolezen import (
    ALONE, EDGES, FAR, FAR_LENGTH, FAR_PLACE, LAST, SHARP, edge_case, edge_tokens, greedy, key_that_matters, through_slots, tokens_with,
)

pytestmark = pytest.mark.gpu

DTYPES = ["float32", "bfloat16"]

# sizes the matrix-core kernels take (heads of 64, 80 and 128, latent rows of 160; projections read as they lie, and widened
# ones) beside the odd ones of the others; chunks and windows that cross steps of 32 keys and pages
WIDE = cases.config_of(
    [
        (cases.attention(heads=8, kv_heads=2, dim=128, vdim=128, chunk=70, scale=0.09), 384),
        (cases.latent(heads=4, dim=32, rot_dim=32, vdim=64, q_rank=96, kv_rank=128, scale=0.12, window=45), 256),
        (cases.attention(heads=4, kv_heads=2, dim=128, vdim=128, chunk=52, scale=0.1, kv_from=0), 128),
        (cases.attention(heads=3, kv_heads=3, dim=48, vdim=80, chunk=33, scale=0.15), 96),
        (cases.latent(heads=2, dim=64, rot_dim=16, vdim=32, q_rank=64, kv_rank=96, scale=0.12, window=130, dims=8), None),
        (cases.attention(heads=6, kv_heads=3, dim=48, vdim=80, chunk=99, scale=0.12, kv_from=3), 200),
    ],
    vocab=300, width=288, scale=4.0,
)


@pytest.fixture(scope="module")
def kernels():
    from llmserve_amd.kernels import HipKernels

    return {"float32": HipKernels(torch.float32), "bfloat16": HipKernels(torch.bfloat16)}


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    root = tmp_path_factory.mktemp("dolezen_gpu")
    return {
        "mixed": cases.write_folder(root / "mixed", cases.MIXED, seed=7),
        "sharp": cases.write_folder(root / "sharp", SHARP, seed=11, sharp=True),
        "wide": cases.write_folder(root / "wide", WIDE, seed=13),
    }


def runner_for(folder, kernels, dtype, page=16, pages=64, slots=4, longest=None):
    loaded = load_model_folder(folder, dtype)
    return ModelRunner(loaded, kernels[dtype], CacheConfig(block_size=page, num_blocks=pages, max_sequences=slots), max_sequence_length=longest)


def agree(got, want, dtype):
    """float32: element by element.  bfloat16: the error of a row, mean taken off, is small beside the row's own spread."""
    got, want = got.float(), want.float()
    if dtype == "float32":
        torch.testing.assert_close(got, want, atol=1e-3, rtol=1e-3)
        return
    error = (got - want) - (got - want).mean(-1, keepdim=True)
    spread = want - want.mean(-1, keepdim=True)
    ratio = error.pow(2).mean(-1).sqrt() / spread.pow(2).mean(-1).sqrt()
    assert float(ratio.max()) < 0.06, f"a bfloat16 row differs by {float(ratio.max()):.3f} of its spread"


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(ALONE))
def test_each_mechanism_layer_by_layer(tmp_path, kernels, dtype, name):
    folder = cases.write_folder(tmp_path / "m", ALONE[name], seed=len(name))
    config, tensors = plain.read_folder(folder)
    tokens = cases.tokens_of(67, config["vocab"], seed=5)
    want, want_streams = plain.forward(config, tensors, tokens)
    loaded = load_model_folder(folder, dtype)
    runner = ModelRunner(loaded, kernels[dtype], CacheConfig(block_size=8, num_blocks=16, max_sequences=2), use_graphs=False)
    seen = []
    runner.model.observer = lambda index, hidden, delta: seen.append((hidden + (delta if delta.ndim == 2 else delta.sum(0))).cpu())
    logits = runner.step([StepEntry("a", tokens, range(len(tokens)))], create_missing=True).float().cpu()
    for got, stream in zip(seen, want_streams, strict=True):
        agree(got, stream, dtype)
    agree(logits, want, dtype)
    runner.close()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("which", ["mixed", "sharp", "wide"])
def test_whole_then_one_by_one_then_portions(folders, kernels, dtype, which):
    if which == "sharp" and dtype == "bfloat16":
        pytest.skip("attention that looks at one key amplifies rounding: this model is for the 32-bit run")
    folder = folders[which]
    config, tensors = plain.read_folder(folder)
    tokens = cases.tokens_of(150, config["vocab"], seed=3)
    want, _ = plain.forward(config, tensors, tokens)
    runner = runner_for(folder, kernels, dtype, page=16, pages=40)
    prompts = {"whole": tokens, "tail": tokens, "cut": tokens, "pairs": tokens[:40]}
    got = cases.run_steps(runner, [[("whole", 150)]], prompts)
    agree(torch.stack([got[("whole", p)] for p in range(150)]), want, dtype)
    got = cases.run_steps(runner, [[("tail", 61)]] + [[("tail", 1)]] * 89, prompts)
    agree(torch.stack([got[("tail", p)] for p in range(150)]), want, dtype)
    sizes = [7, 2, 16, 3, 2, 1, 25, 1, 14, 2, 2, 9, 33, 2, 31]
    got = cases.run_steps(runner, [[("cut", n)] for n in sizes], prompts)
    agree(torch.stack([got[("cut", p)] for p in range(150)]), want, dtype)
    got = cases.run_steps(runner, [[("pairs", 2)]] * 20, prompts)
    agree(torch.stack([got[("pairs", p)] for p in range(40)]), want[:40], dtype)
    assert runner.cache.used_pages == 0
    runner.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_pages_behind_a_chunk_or_a_window_are_given_back(tmp_path, kernels, dtype):
    values = cases.config_of([(cases.attention(chunk=14), 8), (cases.latent(window=11), None), (cases.attention(heads=2, chunk=21, kv_from=0), 16),
                              (cases.attention(heads=2, kv_heads=1, dim=40, vdim=8, chunk=12), None)])
    folder = cases.write_folder(tmp_path / "m", values, seed=3)
    config, tensors = plain.read_folder(folder)
    tokens = cases.tokens_of(260, 67, seed=9)
    want, _ = plain.forward(config, tensors, tokens)
    runner = runner_for(folder, kernels, dtype, page=8, pages=10, longest=512)  # 80 tokens' room a group for 260
    got = cases.run_steps(runner, [[("long", 20)]] * 11 + [[("long", 1)]] * 40, {"long": tokens})
    agree(torch.stack([got[("long", p)] for p in range(260)]), want, dtype)
    runner.close()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("which", ["mixed", "wide"])
def test_mixed_batches_with_pages_and_slots_used_again(folders, kernels, dtype, which):
    folder = folders[which]
    config, tensors = plain.read_folder(folder)
    lengths = {"a": 45, "b": 9, "c": 30, "d": 61, "e": 1, "f": 26, "g": 40}
    prompts = {name: cases.tokens_of(n, config["vocab"], seed=20 + n) for name, n in lengths.items()}
    want = {name: plain.forward(config, tensors, prompts[name])[0] for name in prompts}
    runner = runner_for(folder, kernels, dtype, page=8, pages=16, slots=3)
    rows = [(row, want[name][position]) for _, got in through_slots(runner, lengths, prompts, page=8, pages=16) for (name, position), row in got.items()]
    agree(torch.stack([row for row, _ in rows]), torch.stack([row for _, row in rows]), dtype)
    assert runner.cache.used_pages == 0 and len(runner.cache.sequences) == 0
    assert runner.step_counts["replayed"] > 0  # steps of one shape came back and were replayed from their graph
    runner.close()


@pytest.mark.parametrize("kind", list(EDGES))
def test_one_key_just_inside_and_just_outside(tmp_path, kernels, kind):
    folder, asker, key = edge_case(tmp_path, kind)
    config, tensors = plain.read_folder(folder)
    inside, outside = EDGES[kind]
    for place in inside + outside[:2]:
        tokens = edge_tokens(place, key, asker) + [asker]
        want, _ = plain.forward(config, tensors, tokens)
        for page in (8, 16):
            runner = runner_for(folder, kernels, "float32", page=page, pages=40)
            got = cases.run_steps(runner, [[("p", LAST + 2)]], {"p": tokens})
            agree(torch.stack([got[("p", LAST)], got[("p", LAST + 1)]]), want[-2:], "float32")
            got = cases.run_steps(runner, [[("d", 50)], [("d", 11)], [("d", 2)]] + [[("d", 1)]] * (LAST - 61), {"d": tokens})
            agree(torch.stack([got[("d", LAST)], got[("d", LAST + 1)]]), want[-2:], "float32")
            runner.close()


@pytest.mark.parametrize("name", list(FAR))
def test_a_key_far_back(tmp_path, kernels, name):
    folder, asker, key = key_that_matters(tmp_path, FAR[name], FAR_LENGTH, (FAR_PLACE,))
    config, tensors = plain.read_folder(folder)
    tokens = tokens_with(FAR_LENGTH, FAR_PLACE, key, asker)
    want, _ = plain.forward(config, tensors, tokens)
    runner = runner_for(folder, kernels, "float32", page=16, pages=40)
    got = cases.run_steps(runner, [[("p", FAR_LENGTH)]], {"p": tokens})
    agree(got[("p", FAR_LENGTH - 1)][None], want[-1][None], "float32")
    got = cases.run_steps(runner, [[("d", 333)], [("d", 47)]] + [[("d", 1)]] * 10, {"d": tokens})
    agree(got[("d", FAR_LENGTH - 1)][None], want[-1][None], "float32")
    runner.close()


def test_greedy_generation_through_the_engine(folders, kernels):
    config, tensors = plain.read_folder(folders["mixed"])
    prompts = [cases.tokens_of(n, 67, seed=40 + n) for n in (1, 6, 17, 30)]
    expected = [greedy(config, tensors, prompt, 12) for prompt in prompts]
    runner = runner_for(folders["mixed"], kernels, "float32", page=16, pages=32, slots=4)
    core = EngineCore(runner, SchedulerConfig(max_batch_size=3, max_tokens_per_step=24), prefill_chunk_size=8)
    assert core.generate(prompts, GenerationConfig(max_new_tokens=12)) == expected
    assert runner.cache.used_pages == 0
    runner.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_trace_replay(folders, tmp_path, dtype):
    """bin/trace_run: portions beside single tokens, a request that pauses, slots used again."""
    config, tensors = plain.read_folder(folders["wide"])
    prompts = {name: cases.tokens_of(n, config["vocab"], seed=n) for name, n in {"a": 110, "b": 23, "c": 5, "d": 33, "e": 64}.items()}
    want = {name: plain.forward(config, tensors, tokens)[0] for name, tokens in prompts.items()}
    trace = TraceBuilder()
    trace.step([("a", prompts["a"][:40]), ("b", prompts["b"][:2])])
    trace.step([("a", prompts["a"][40:41]), ("b", prompts["b"][2:20]), ("c", prompts["c"])], end=["c"])
    trace.step([("a", prompts["a"][41:42]), ("d", prompts["d"][:30])])
    trace.step([("b", prompts["b"][20:]), ("a", prompts["a"][42:]), ("d", prompts["d"][30:31])], end=["a", "b"])
    trace.step([("d", prompts["d"][31:32]), ("e", prompts["e"])], end=["e"])
    trace.step([("d", prompts["d"][32:])], end=["d"])
    found = trace.collect(replay(folders["wide"], dtype, trace.steps, tmp_path / "out", max_tokens=256, block_size=16, vocab=config["vocab"]))
    assert len(found) == sum(len(tokens) for tokens in prompts.values())
    keys = sorted(found)
    agree(torch.stack([found[key] for key in keys]), torch.stack([want[name][position] for name, position in keys]), dtype)
