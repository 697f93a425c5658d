"""The Dubesun decoder through the engine's loader, cache manager and step function (over the torch stand-in of the
kernel library, on the CPU) against the plain implementation: mechanism by mechanism, and through schedules of steps."""

from __future__ import annotations

import json
import math

import pytest
import torch

from llmserve_amd import CacheConfig, EngineCore, GenerationConfig, ModelRunner, SchedulerConfig, StepEntry
from llmserve_amd.cache.pool import CacheFullError
from llmserve_amd.config import ConfigError
from llmserve_amd.config.dubesun import DubesunConfig
from llmserve_amd.parts import DistanceBuckets, FixedState, LayerRun, PagedKeyValue
from llmserve_amd.weights import load_model_folder
from tests import dubesun_cases as cases
from tests.plain import dubesun_plain as plain
from tests.test_dolezen import through_slots
from tests.torch_kernels import TorchKernels


def runner_for(folder, page=4, pages=64, slots=4, dtype="float32"):
    loaded = load_model_folder(folder, dtype)
    return ModelRunner(loaded, TorchKernels(loaded.dtype), CacheConfig(block_size=page, num_blocks=pages, max_sequences=slots), use_graphs=False)


def oracle(folder, tokens):
    config, tensors = plain.read_folder(folder)
    logits, streams = plain.forward(config, tensors, tokens)
    return logits.float(), streams.float()


def close(got, want, atol=3e-4):
    torch.testing.assert_close(got.float(), want.float(), atol=atol, rtol=3e-4)


# ---------------------------------------------------------------------------- configuration and weights


def test_config_round_trip_and_refusals():
    config = DubesunConfig.from_dict(cases.MIXED)
    assert DubesunConfig.from_dict(config.to_config_json()) == config
    assert json.loads(json.dumps(config.to_config_json())) == cases.MIXED
    assert config.max_position_embeddings == 512
    bare = cases.config_of([(cases.difference(conv=None, coef=None), None), (cases.biased(), None)])
    del bare["layers"][0]["mixer"]["kv_heads"], bare["layers"][0]["mlp"], bare["layers"][1]["mixer"]["vdim"], bare["layers"][1]["mixer"]["buckets"]
    read = DubesunConfig.from_dict(bare)
    assert (read.layers[0].mixer.kv_heads, read.layers[0].mixer.conv, read.layers[0].mixer.temperature, read.layers[0].mlp) == (6, None, None, None)
    assert read.layers[1].mixer.buckets is None
    assert read.with_sizes_of({"l1.mix.rel": (14, 4)}).layers[1].mixer.buckets == 14
    assert DubesunConfig.from_dict(read.to_config_json()) == read
    with pytest.raises(ConfigError, match="buckets"):  # a model without tensors has to say how many
        from llmserve_amd.models.dubesun import dubesun_spec

        dubesun_spec(read)
    broken = [
        cases.config_of([(cases.difference(heads=5, kv_heads=2), None)]),  # heads no multiple of kv_heads
        cases.config_of([(cases.difference(kv_from=0), None)]),  # its own keys and values, which it does not make
        cases.config_of([(cases.difference(), None), (cases.difference(kv_from=2), None), (cases.difference(), None)]),  # of a later layer
        cases.config_of([(cases.biased(), None), (cases.difference(kv_from=0), None)]),  # of a layer of another kind
        cases.config_of([(cases.difference(), None), (cases.difference(kv_from=0), None), (cases.difference(kv_from=1), None)]),  # of one that has none
        cases.config_of([(cases.difference(), None), (cases.difference(dim=16, kv_from=0), None)]),  # of other sizes
        cases.config_of([(cases.difference(), None), (cases.difference(kv_heads=3, kv_from=0), None)]),
        cases.config_of([(cases.difference(every=0), None)]),
        cases.config_of([(cases.difference(conv=0), None)]),
        cases.config_of([(cases.biased(bias_max=5, buckets=10), None)]),  # the last bucket begins before the first half ends
        cases.config_of([(cases.biased(), cases.experts(3, 4))]),  # more experts a token than there are
        cases.config_of([(cases.biased(), cases.experts(limit=0.0))]),
        cases.config_of([({"type": "window", "mixer": {}}, None)]),
        cases.config_of([]),
    ]
    missing = cases.config_of([(cases.difference(), None)])
    del missing["layers"][0]["mixer"]["diff"]
    other = cases.config_of([(cases.difference(), cases.experts())])
    other["layers"][0]["mlp"]["kind"] = "dense"
    narrow = cases.config_of([(cases.biased(), None)])
    narrow["layers"][0]["mixer"]["vdim"] = 16  # the values are the keys
    for values in broken + [missing, other, narrow, {**cases.MIXED, "max_positions": None}]:
        with pytest.raises(ConfigError):
            DubesunConfig.from_dict(values)


def test_folder_names_and_what_each_run_keeps(tmp_path):
    from llmserve_amd.models.dubesun import dubesun_spec

    spec = dubesun_spec(DubesunConfig.from_dict(cases.MIXED))
    names = set(spec.tensors())
    assert {"embed", "pos", "head", "final.norm", "l0.norm1", "l0.mix.q.conv", "l0.mix.k.conv", "l0.mix.v.conv", "l0.mix.q.norm", "l0.mix.k.norm",
            "l0.mix.lq1", "l0.mix.lk2", "l0.mlp.router", "l0.mlp.e4.gate", "l1.mix.q.b", "l1.mix.k.b", "l1.mix.rel", "l1.mix.g", "l3.mix.q.conv", "l3.mix.q.norm"} <= names
    assert not {"l0.norm2", "l0.mix.q.b", "l1.mix.v", "l1.mix.v.b", "l1.mix.q.norm", "l1.mlp.router", "l3.mix.k", "l3.mix.v", "l3.mix.k.conv",
                "l3.mix.k.norm", "l5.mix.q.conv", "l0.mlp.router.b"} & names
    assert [(run.layer, run.reads) for run in spec.run_order] == [(0, None), (1, None), (2, None), (3, 0), (4, None), (5, 2)]
    # a key row holds both maps beside a value row of the same width; a reader keeps the inputs of its own convolution alone
    assert spec.cell_need(0) == {"keys": PagedKeyValue(2, 64), "window": FixedState((3, 2 * 6 * 24 + 2 * 2 * 24 + 2 * 40))}
    assert spec.cell_need(3) == {"keys": PagedKeyValue(2, 64), "window": FixedState((5, 2 * 2 * 24))}
    assert spec.cell_need(2)["keys"] == PagedKeyValue(1, 32) and spec.cell_need(5) == {"keys": PagedKeyValue(1, 32)}
    assert spec.cell_need(1) == PagedKeyValue(2, 16)
    runner = runner_for(cases.write_folder(tmp_path / "m", cases.MIXED))
    cells = runner.cells
    assert cells[3]["keys"].keys.data_ptr() == cells[0]["keys"].keys.data_ptr() and not cells[3]["keys"].writable and cells[0]["keys"].writable
    assert cells[3]["window"].writable and cells[3]["window"].state.data_ptr() != cells[0]["window"].state.data_ptr()
    assert sorted(len(group.cells) for group in runner.cache.groups) == [1, 1, 1, 1] and len(runner.cache.states) == 3
    for extra in ("l3.mix.k", "l1.mix.v"):
        tensors = cases.random_tensors(cases.MIXED, 3)
        tensors[extra] = torch.ones((8, 40), dtype=torch.bfloat16)
        with pytest.raises(Exception, match=extra):
            load_model_folder(cases.write_folder(tmp_path / extra, cases.MIXED, tensors=tensors), "float32")


def test_runs_that_read_a_part_of_another_cell(tmp_path):
    from dataclasses import replace

    from llmserve_amd.models.dubesun import dubesun_spec

    spec = dubesun_spec(DubesunConfig.from_dict(cases.MIXED))
    assert spec.run_order[3].takes("keys") and not spec.run_order[3].takes("window") and not spec.run_order[0].takes("keys")
    with pytest.raises(ValueError, match="reads none"):
        replace(spec, run_order=(LayerRun(0, reads_only=("keys",)),))
    with pytest.raises(ValueError, match="different caches"):  # the whole cell, whose convolutions are not the reader's
        replace(spec, run_order=tuple(replace(run, reads_only=None) for run in spec.run_order))
    with pytest.raises(ValueError, match="different caches"):
        replace(spec, run_order=(LayerRun(0), LayerRun(2), LayerRun(3, reads=1, reads_only=("keys",))))


def test_a_request_is_no_longer_than_the_table_of_positions(tmp_path):
    values = cases.config_of([(cases.biased(), None)], max_positions=21)
    runner = runner_for(cases.write_folder(tmp_path / "m", values))
    tokens = cases.tokens_of(22, 67, seed=1)
    runner.step([StepEntry("a", tokens[:21], [])], create_missing=True)
    with pytest.raises(CacheFullError):
        runner.step([StepEntry("a", tokens[21:], [0])])
    core = EngineCore(runner_for(tmp_path / "m"), SchedulerConfig(max_batch_size=2, max_tokens_per_step=24))
    with pytest.raises(Exception):  # (a prompt and its answer that do not fit the positions)
        core.generate([tokens[:15]], GenerationConfig(max_new_tokens=12))


# ---------------------------------------------------------------------------- distances

BUCKETS = [(2, 3), (4, 9), (10, 37), (10, 512), (22, 90), (32, 128), (32, 1000), (33, 200), (64, 70)]


@pytest.mark.parametrize("buckets,furthest", BUCKETS)
def test_buckets_of_distances(buckets, furthest):
    table = DistanceBuckets(buckets, float(furthest))
    found = [table.of(distance) for distance in range(3 * furthest)]
    assert found == [plain.distance_bucket(distance, buckets, furthest) for distance in range(3 * furthest)]
    assert found[: buckets // 2] == list(range(buckets // 2)) and found[furthest] == buckets - 1 and sorted(found) == found
    assert found[table.reach - 1] == buckets - 1 and (table.reach == 1 or found[table.reach - 2] < buckets - 1)
    assert table.by_distance().tolist() == found[: table.reach]


def test_a_bucket_begins_exactly_where_its_power_lies():
    """half 4, four later buckets up to 64: they begin at 4 * 16^(k / 4), exactly 4, 8, 16 and 32."""
    table = DistanceBuckets(8, 64.0)
    assert [table.of(n) for n in (3, 4, 7, 8, 15, 16, 31, 32, 33, 63, 64, 1000)] == [3, 4, 4, 5, 5, 6, 6, 7, 7, 7, 7, 7]
    assert table.reach == 33
    for buckets, furthest in ((1, 9.0), (10, 5.0)):
        with pytest.raises(ValueError):
            DistanceBuckets(buckets, furthest)


# ---------------------------------------------------------------------------- every mechanism alone

ALONE = {
    "difference": cases.config_of([(cases.difference(), None)]),
    "difference, as many kv heads as heads, maps wider than values": cases.config_of([(cases.difference(heads=3, kv_heads=3, dim=40, vdim=8), cases.experts())]),
    "difference, values twice as wide as a map": cases.config_of([(cases.difference(heads=4, kv_heads=2, dim=16, vdim=32, conv=3), cases.experts())]),
    "difference, no convolution": cases.config_of([(cases.difference(conv=None), None)]),
    "difference, a convolution of one tap": cases.config_of([(cases.difference(conv=1, dim=10, vdim=12), None)]),
    "difference, seven taps": cases.config_of([(cases.difference(heads=2, kv_heads=1, dim=16, vdim=16, conv=7), None)]),
    "difference, no temperature": cases.config_of([(cases.difference(coef=None, diff=0.8), None)]),
    "difference, odd sizes": cases.config_of([(cases.difference(heads=3, kv_heads=1, dim=5, vdim=7, conv=2), cases.experts(3, 2, 5))]),
    "difference over another layer's keys": cases.config_of([(cases.difference(), None), (cases.difference(heads=2, conv=2, kv_from=0), cases.experts())]),
    "two readers of one layer, one without a convolution": cases.config_of(
        [(cases.difference(conv=None), None), (cases.biased(), None), (cases.difference(heads=8, conv=3, kv_from=0), None), (cases.difference(heads=2, conv=None, kv_from=0), None)]),
    "bias by distance": cases.config_of([(cases.biased(), None)]),
    "bias by distance, few buckets": cases.config_of([(cases.biased(heads=2, kv_heads=1, dim=16, bias_max=3, buckets=4), cases.experts())]),
    "bias by distance, as many kv heads as heads, odd sizes": cases.config_of([(cases.biased(heads=3, kv_heads=3, dim=11, bias_max=200, buckets=12), None)]),
    "experts, one a token": cases.config_of([(cases.biased(), cases.experts(6, 1, 16))]),
    "experts, all of them": cases.config_of([(cases.biased(), cases.experts(4, 4, 17, limit=0.2))]),
}


@pytest.mark.parametrize("name", list(ALONE))
def test_each_mechanism_layer_by_layer(tmp_path, name):
    folder = cases.write_folder(tmp_path / "m", ALONE[name], seed=len(name))
    tokens = cases.tokens_of(47, ALONE[name]["vocab"], seed=5)
    want_logits, want_streams = oracle(folder, tokens)
    runner = runner_for(folder)
    seen = []
    runner.model.observer = lambda index, hidden, delta: seen.append(hidden + (delta if delta.ndim == 2 else delta.sum(0)))
    logits = runner.step([StepEntry("a", tokens, range(len(tokens)))], create_missing=True)
    assert len(seen) == want_streams.shape[0]
    for index, stream in enumerate(seen):
        close(stream, want_streams[index])
    close(logits, want_logits)


def test_every_mechanism_matters(tmp_path):
    """The plain implementation without one of them gives other logits: the comparisons here would see one left out."""
    folder = cases.write_folder(tmp_path / "m", cases.MIXED, seed=4)
    config, tensors = plain.read_folder(folder)
    tokens = cases.tokens_of(60, 67, seed=1)
    want, _ = plain.forward(config, tensors, tokens)

    def changed(path, value):
        other = json.loads(json.dumps(config))
        at = other
        for key in path[:-1]:
            at = at[key]
        at[path[-1]] = value
        return plain.forward(other, tensors, tokens)[0]

    def with_tensor(name, value):
        return plain.forward(config, dict(tensors, **{name: value}), tokens)[0]

    def last_tap_alone(name):
        taps = torch.zeros_like(tensors[name])
        taps[:, -1] = tensors[name][:, -1]
        return taps

    others = {
        "a score's scale": changed(("layers", 0, "mixer", "scale"), 0.29),
        "a reader's scale": changed(("layers", 3, "mixer", "scale"), 0.23),
        "the constant of the difference": changed(("layers", 3, "mixer", "diff"), 0.35),
        "the temperature's coefficient": changed(("layers", 3, "mixer", "q_temp", "coef"), 0.6),
        "how often the temperature changes": changed(("layers", 0, "mixer", "q_temp", "every"), 6),
        "where the last bucket begins": changed(("layers", 1, "mixer", "bias_max"), 44),
        "the experts' limit": changed(("layers", 2, "mlp", "expert", "limit"), 0.5),
        "the experts a token": changed(("layers", 4, "mlp", "router", "top"), 2),
        "the positions": with_tensor("pos", torch.zeros_like(tensors["pos"])),
        "a norm's weight": with_tensor("l0.norm1", torch.zeros_like(tensors["l0.norm1"])),
        "the last norm's weight": with_tensor("final.norm", torch.zeros_like(tensors["final.norm"])),
        "the queries' norm": with_tensor("l3.mix.q.norm", torch.ones_like(tensors["l3.mix.q.norm"])),
        "the keys' norm": with_tensor("l0.mix.k.norm", torch.ones_like(tensors["l0.mix.k.norm"])),
        "lambda": with_tensor("l2.mix.lq1", torch.zeros_like(tensors["l2.mix.lq1"])),
        "the biases by distance": with_tensor("l4.mix.rel", torch.zeros_like(tensors["l4.mix.rel"])),
        "the gate": with_tensor("l4.mix.g", torch.zeros_like(tensors["l4.mix.g"])),
        "the bias of q": with_tensor("l1.mix.q.b", torch.zeros_like(tensors["l1.mix.q.b"])),
        "the bias of k": with_tensor("l1.mix.k.b", torch.zeros_like(tensors["l1.mix.k.b"])),
    }
    for name in ("l0.mix.q", "l0.mix.k", "l0.mix.v", "l3.mix.q"):
        others[f"the convolution of {name}"] = with_tensor(name + ".conv", last_tap_alone(name + ".conv"))
    for name, other in others.items():
        assert float((other - want).abs().max()) > 0.01, name


def test_experts_take_the_mixers_result_along(tmp_path):
    """The block hands the mixer's rows to the experts, whose last kernel adds them; apart, a kernel adds the two."""
    folder = cases.write_folder(tmp_path / "m", cases.MIXED, seed=3)
    tokens = cases.tokens_of(30, 67, seed=5)
    along, apart = runner_for(folder), runner_for(folder)
    for layer in apart.model.layers:
        if layer.feed_forward is not None:
            assert layer.feed_forward.adds_beside
            layer.feed_forward.adds_beside = False
    want = along.step([StepEntry("a", tokens, range(30))], create_missing=True)
    close(apart.step([StepEntry("a", tokens, range(30))], create_missing=True), want)


# ---------------------------------------------------------------------------- steps and cache


@pytest.fixture(scope="module")
def mixed_folder(tmp_path_factory):
    return cases.write_folder(tmp_path_factory.mktemp("dubesun") / "mixed", cases.MIXED, seed=7)


SHARP = cases.config_of(
    [(cases.difference(heads=2, kv_heads=1, dim=8, vdim=16, scale=1.6, conv=3), cases.experts(3, 2, 16)),
     (cases.biased(heads=2, kv_heads=1, dim=8, scale=2.0, bias_max=100, buckets=16), None),
     (cases.difference(heads=3, kv_heads=1, dim=8, vdim=16, scale=1.9, conv=5, kv_from=0), None)],
    vocab=43, width=24,
)


@pytest.fixture(scope="module")
def sharp_folder(tmp_path_factory):
    """Attention that looks at one key, wherever it is."""
    return cases.write_folder(tmp_path_factory.mktemp("dubesun") / "sharp", SHARP, seed=11)


@pytest.mark.parametrize("which", ["mixed", "sharp"])
def test_whole_then_one_by_one_then_portions(mixed_folder, sharp_folder, which):
    folder = mixed_folder if which == "mixed" else sharp_folder
    vocab = plain.read_folder(folder)[0]["vocab"]
    tokens = cases.tokens_of(150, vocab, seed=3)
    want, _ = oracle(folder, tokens)
    runner = runner_for(folder, page=8, pages=80)
    prompts = {"whole": tokens, "tail": tokens, "cut": tokens, "pairs": tokens[:40]}
    got = cases.run_steps(runner, [[("whole", 150)]], prompts)
    close(torch.stack([got[("whole", p)] for p in range(150)]), want, atol=1e-3)
    got = cases.run_steps(runner, [[("tail", 61)]] + [[("tail", 1)]] * 89, prompts)  # long decoding
    close(torch.stack([got[("tail", p)] for p in range(150)]), want, atol=1e-3)
    sizes = [7, 2, 16, 3, 2, 1, 25, 1, 14, 2, 2, 9, 33, 2, 31]
    assert sum(sizes) == 150
    got = cases.run_steps(runner, [[("cut", n)] for n in sizes], prompts)
    close(torch.stack([got[("cut", p)] for p in range(150)]), want, atol=1e-3)
    got = cases.run_steps(runner, [[("pairs", 2)]] * 20, prompts)
    close(torch.stack([got[("pairs", p)] for p in range(40)]), want[:40], atol=1e-3)
    assert runner.cache.used_pages == 0


def test_the_first_tokens_of_a_sequence(mixed_folder):
    """Prompts of one to seven tokens, whole and token by token, in slots that others used: convolutions before the start."""
    runner = runner_for(mixed_folder, slots=1)
    for length in (1, 2, 3, 5, 7):
        tokens = cases.tokens_of(length, 67, seed=length)
        want, _ = oracle(mixed_folder, tokens)
        got = cases.run_steps(runner, [[("w", length)]], {"w": tokens})
        close(torch.stack([got[("w", p)] for p in range(length)]), want)
        got = cases.run_steps(runner, [[("s", 1)]] * length, {"s": tokens})
        close(torch.stack([got[("s", p)] for p in range(length)]), want)


@pytest.mark.parametrize("which", ["mixed", "sharp"])
def test_mixed_batches_with_pages_and_slots_used_again(mixed_folder, sharp_folder, which):
    """Six unequal requests through three slots and a small pool: portions beside single tokens, requests that pause for
    a step, slots and pages taken over from requests that ended."""
    folder = mixed_folder if which == "mixed" else sharp_folder
    vocab = plain.read_folder(folder)[0]["vocab"]
    lengths = {"a": 45, "b": 9, "c": 30, "d": 61, "e": 1, "f": 26}
    prompts = {name: cases.tokens_of(n, vocab, seed=20 + n) for name, n in lengths.items()}
    want = {name: oracle(folder, prompts[name])[0] for name in prompts}
    runner = runner_for(folder, page=4, pages=30, slots=3)
    for step, got in through_slots(runner, lengths, prompts, page=4, pages=30):
        for (name, position), row in got.items():
            close(row, want[name][position], atol=1e-3)
    assert runner.cache.used_pages == 0 and len(runner.cache.sequences) == 0


# ---------------------------------------------------------------------------- one key

NEAR, FAR = 78, 390  # tokens of a short and of a long prompt, the last one asking
PLACES = {NEAR: (76, 64, 63, 48, 1), FAR: (7, 16, 300)}  # next to the query, at pages' borders, at the start; hundreds back


def tokens_with(length, place, token, asker):
    tokens = [1 + (i % 30) for i in range(length)]
    tokens[place], tokens[-1] = token, asker
    return tokens


KEYED = {
    # (no convolution: it would bring the neighbours' tokens into the one key; the schedules above have them)
    "difference": cases.difference(heads=2, kv_heads=1, dim=16, vdim=8, scale=1.5, conv=None, coef=0.1, every=50),
    "bias": cases.biased(heads=2, kv_heads=1, dim=16, scale=1.5, bias_max=100, buckets=16),
}


def key_that_matters(folder_root, kind, length):
    """A one-layer model whose scores are large, and two tokens (asker, key) such that the last query's answer, the asker's,
    hangs on the one key at any of the places: found by trying seeds and pairs on the plain implementation."""
    values = cases.config_of([(KEYED[kind], None)], vocab=37, width=24)
    for seed in range(1, 60):
        tensors = cases.random_tensors(values, seed)
        tensors["pos"] = tensors["pos"] * 0.05  # (a key is recognised by its token, wherever it stands)
        if "l0.mix.rel" in tensors:
            tensors["l0.mix.rel"] = tensors["l0.mix.rel"] * 0.3
        folder = cases.write_folder(folder_root / f"{kind}{seed}", values, tensors=tensors)
        config, read = plain.read_folder(folder)
        for asker in range(31, 37):
            for key in range(31, 37):
                if asker == key:
                    continue
                for place in PLACES[length]:
                    one, other = (plain.forward(config, read, tokens_with(length, place, token, asker))[0][-1] for token in (key, 30))
                    if float((one - other).abs().max()) < 0.2:
                        break
                else:
                    return folder, asker, key
    raise AssertionError("no seed gave a key that matters at every place")


@pytest.mark.parametrize("length", [NEAR, FAR])
@pytest.mark.parametrize("kind", list(KEYED))
def test_one_key(tmp_path, kind, length):
    """A query whose answer hangs on one key: next to it, at pages' borders, at the start, hundreds of tokens back; in a
    prompt's portion and decoded alone, with pages of 4 and of 16."""
    folder, asker, key = key_that_matters(tmp_path, kind, length)
    config, tensors = plain.read_folder(folder)
    for place in PLACES[length]:
        tokens = tokens_with(length, place, key, asker)
        want, _ = plain.forward(config, tensors, tokens)
        for page in (4, 16):
            runner = runner_for(folder, page=page, pages=-(-length // page) + 3)
            got = cases.run_steps(runner, [[("p", length)]], {"p": tokens})
            close(got[("p", length - 1)], want[-1].float(), atol=1e-3)
            got = cases.run_steps(runner, [[("d", length - 15)], [("d", 2)], [("d", 3)]] + [[("d", 1)]] * 10, {"d": tokens})
            close(got[("d", length - 1)], want[-1].float(), atol=1e-3)


def test_a_bias_just_inside_and_just_outside_a_bucket(tmp_path):
    """One bucket's bias towers over the others: the query sees the keys at that bucket's distances alone, so its first and
    last distance show, at every position and in decoding."""
    buckets, furthest = 12, 70
    values = cases.config_of([(cases.biased(heads=2, kv_heads=1, dim=16, scale=0.2, bias_max=furthest, buckets=buckets), None)])
    tensors = cases.random_tensors(values, 5)
    for bucket in (0, 4, 6, 9, buckets - 1):
        tensors["l0.mix.rel"] = torch.zeros((buckets, 2), dtype=torch.bfloat16)
        tensors["l0.mix.rel"][bucket] = 30.0
        folder = cases.write_folder(tmp_path / str(bucket), values, tensors=tensors)
        tokens = cases.tokens_of(100, 67, seed=bucket)
        want, _ = oracle(folder, tokens)
        first = next(d for d in range(200) if plain.distance_bucket(d, buckets, furthest) == bucket)
        read, asked = plain.read_folder(folder), 99
        for distance, matters in ((first, True), (first - 1, False)):
            if distance < 0:
                continue
            moved = list(tokens)
            moved[asked - distance] = (moved[asked - distance] + 1) % 67
            if distance == 0:
                continue
            other = plain.forward(*read, moved)[0][asked].float()
            effect = float((other - want[asked]).abs().max())
            assert effect > 1e-3 if matters else effect < 1e-6, (bucket, distance, effect)
        runner = runner_for(folder, page=8, pages=16)
        got = cases.run_steps(runner, [[("p", 100)]], {"p": tokens})
        close(torch.stack([got[("p", p)] for p in range(100)]), want)
        got = cases.run_steps(runner, [[("d", 40)], [("d", 2)]] + [[("d", 1)]] * 58, {"d": tokens})
        close(torch.stack([got[("d", p)] for p in range(100)]), want)


def test_the_temperature_steps_between_two_positions():
    """Just before and just behind every multiple of `every`."""
    for coef, every in ((0.5, 7), (0.3, 128), (2.0, 1)):
        grown = plain.query_temperature(3 * every + 1, coef, every)
        for k in (1, 2, 3):
            assert math.isclose(float(grown[k * every - 1]), 1.0 + coef * math.log(k + 1))  # the position p with p + 1 = k every
            assert k == 1 and every == 1 or math.isclose(float(grown[k * every - 2]), 1.0 + coef * math.log(k))


# ---------------------------------------------------------------------------- generation


def greedy(config, tensors, prompt, count):
    tokens = list(prompt)
    for _ in range(count):
        tokens.append(int(torch.argmax(plain.forward(config, tensors, tokens)[0][-1])))
    return tokens[len(prompt):]


def test_greedy_generation_through_the_engine(mixed_folder):
    config, tensors = plain.read_folder(mixed_folder)
    prompts = [cases.tokens_of(n, 67, seed=40 + n) for n in (1, 6, 17, 30)]
    expected = [greedy(config, tensors, prompt, 7) for prompt in prompts]
    runner = runner_for(mixed_folder, page=4, pages=64, slots=4)
    core = EngineCore(runner, SchedulerConfig(max_batch_size=3, max_tokens_per_step=24), prefill_chunk_size=8)
    assert core.generate(prompts, GenerationConfig(max_new_tokens=7)) == expected
    assert runner.cache.used_pages == 0


def test_the_command_line_writes_a_random_model_folder(tmp_path, capsys):
    """`llmserve random-model` goes through the registry: a Dubesun config.json gives a folder that loads and runs."""
    from llmserve_amd.cli import main

    (tmp_path / "config.json").write_text(json.dumps(cases.MIXED))
    assert main(["random-model", "--config", str(tmp_path / "config.json"), "--output", str(tmp_path / "out"), "--seed", "5", "--std", "0.2"]) == 0
    assert str(tmp_path / "out") in capsys.readouterr().out
    tokens = cases.tokens_of(12, 67, seed=2)
    want, _ = oracle(tmp_path / "out", tokens)
    runner = runner_for(tmp_path / "out")
    close(runner.step([StepEntry("a", tokens, range(12))], create_missing=True), want)
