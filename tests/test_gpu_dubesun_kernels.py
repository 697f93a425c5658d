"""The kernels of the Dubesun parts, each alone against the same operation in elementary float32 torch (the CPU
stand-in of the kernel library), at sizes that are no powers of two and over steps that cut a request's tokens anywhere."""

from __future__ import annotations

import types

import pytest
import torch

from tests.test_gpu_dolezen_kernels import STEPS, attention_case
from tests.test_gpu_sozavik_kernels import DTYPES, close, gpu, step_of
from tests.torch_kernels import TorchKernels

pytestmark = pytest.mark.gpu


@pytest.fixture(scope="module")
def kernels():
    from llmserve_amd.kernels import HipKernels

    return {dtype: HipKernels(dtype) for dtype in DTYPES}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("hidden", [24, 257, 1536])
def test_embedded_rows_with_a_vector_a_position(kernels, dtype, hidden):
    torch.manual_seed(hidden)
    table, places = torch.randn(50, hidden).to(dtype), torch.randn(33, hidden).to(dtype)
    ids, positions = (torch.randint(0, n, (19,), dtype=torch.int32) for n in (50, 33))
    positions[:2] = torch.tensor([0, 32])
    want = TorchKernels(dtype).embedding(table, ids, 1.7, positions=positions, position_table=places)
    got = kernels[dtype].embedding(gpu(table), gpu(ids), 1.7, positions=gpu(positions), position_table=gpu(places))
    close(got, want, torch.float32)
    close(kernels[dtype].embedding(gpu(table), gpu(ids), 1.7), TorchKernels(dtype).embedding(table, ids, 1.7), torch.float32)


# ---------------------------------------------------------------------------- queries, keys and values made ready

HEADS = [
    # heads, kv heads, maps, dim, vdim, width
    (6, 2, 2, 24, 40, 64),
    (12, 2, 2, 64, 128, 128),
    (3, 3, 2, 40, 8, 96),
    (4, 1, 2, 40, 88, 96),
    (2, 1, 2, 5, 7, 32),
    (8, 2, 1, 128, 128, 128),
    (3, 1, 1, 80, 80, 80),
    (5, 5, 1, 11, 11, 16),
    (2, 0, 2, 16, 32, 32),  # queries alone
    (2, 1, 2, 128, 256, 256),
]
CUTS = [([1, 1, 1], [700, 3, 0]), ([33, 1, 7, 2], [0, 90, 250, 3]), ([2, 2, 2], [0, 1, 5]), ([70], [0]), ([1, 1, 1, 1, 1], [0, 1, 2, 3, 4])]


def heads_case(dtype, heads, kv_heads, maps, dim, vdim, width, counts, starts, taps, page, keys_as_values=False):
    from llmserve_amd.cache.cell import CacheCell
    from llmserve_amd.parts import PagedKeyValue

    torch.manual_seed(heads * dim + sum(counts) + (taps or 0))
    q, k, v = heads * maps * dim, kv_heads * maps * dim, 0 if keys_as_values else kv_heads * vdim
    channels, tokens = q + k + v, sum(counts)
    x = torch.randn(tokens, channels + (0 if dim % 8 else 8)).to(dtype)
    tap_rows = torch.randn(channels, taps) if taps else None
    window = torch.randn(len(counts) + 2, taps - 1, channels) if taps and taps > 1 else None
    slots = [len(counts) + 1 - b for b in range(len(counts))]
    if window is not None:
        window[1] = 9.0  # (a slot of nobody in the step)
        for b, start in enumerate(starts):  # what a request of so few tokens has kept: zeros before its start
            window[slots[b], : max(0, taps - 1 - start)] = 0.0
    need = PagedKeyValue(max(kv_heads, 1), width)
    longest = max(s + c for s, c in zip(starts, counts))
    per = -(-longest // page)
    fields = {name: torch.randn(per * len(counts) + 1, *shape).to(dtype) for name, shape in need.page_fields(page).items()}
    tables = (torch.randperm(per * len(counts)) + 1).reshape(len(counts), per).to(torch.int32)
    places = [int(tables[b, p // page]) * page + p % page for b, (s, c) in enumerate(zip(starts, counts)) for p in range(s, s + c)]

    def batch_on(device):
        batch = step_of(counts, starts, slots, device)
        batch.token_sequence = torch.cat([torch.full((c,), b) for b, c in enumerate(counts)]).to(torch.int32).to(device)
        batch.groups = [types.SimpleNamespace(page_size=page, block_tables=tables.to(device), slot_mapping=torch.tensor(places, dtype=torch.int32).to(device), width=per)]
        return batch

    cells = {device: CacheCell(need, group=0, fields={name: value.clone().to(device) for name, value in fields.items()}) for device in ("cpu", "cuda")}
    firsts = (0, q, q if keys_as_values else q + k)
    return x, firsts, tap_rows, window, cells, {device: batch_on(device) for device in cells}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("sizes", HEADS)
@pytest.mark.parametrize("counts,starts", CUTS)
@pytest.mark.parametrize("taps,weighted,temperature", [(4, True, (0.4, 5)), (3, True, None), (2, False, (0.1, 64)), (1, True, (0.7, 1)), (None, True, (0.3, 7)), (6, True, None)])
def test_convolved_heads(kernels, dtype, sizes, counts, starts, taps, weighted, temperature):
    heads, kv_heads, maps, dim, vdim, width = sizes
    x, firsts, tap_rows, window, cells, batches = heads_case(dtype, *sizes, counts, starts, taps, page=8)
    weights = [(1 + 0.3 * torch.randn(dim)).to(dtype) for _ in range(2)] if weighted else [None, None]
    on = lambda t: None if t is None else gpu(t)  # noqa: E731
    windows = {"cpu": None if window is None else window.clone(), "cuda": on(window)}
    options = dict(maps=maps, eps=1e-4, temperature=temperature)
    want = TorchKernels(dtype).convolved_heads(x, *firsts, heads, kv_heads, dim, vdim, width, batches["cpu"], cells["cpu"] if kv_heads else None, taps=tap_rows,
                                               window=windows["cpu"], q_weight=weights[0], k_weight=weights[1], **options)
    got = kernels[dtype].convolved_heads(gpu(x), *firsts, heads, kv_heads, dim, vdim, width, batches["cuda"], cells["cuda"] if kv_heads else None,
                                         taps=on(tap_rows), window=windows["cuda"], q_weight=on(weights[0]), k_weight=on(weights[1]), **options)
    close(got, want, dtype)
    for name in ("keys", "values"):  # what was stored, where; every other entry as it was
        close(cells["cuda"].fields[name], cells["cpu"].fields[name], dtype)
    if window is not None:
        assert torch.equal(windows["cuda"].cpu(), windows["cpu"])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,kv_heads,dim,width", [(8, 2, 128, 128), (4, 2, 24, 32), (3, 3, 11, 16)])
@pytest.mark.parametrize("counts,starts", CUTS)
def test_values_that_are_the_keys(kernels, dtype, heads, kv_heads, dim, width, counts, starts):
    """Queries and keys over their root mean square, and the keys once more as values, as they were."""
    x, firsts, _, _, cells, batches = heads_case(dtype, heads, kv_heads, 1, dim, dim, width, counts, starts, None, page=16, keys_as_values=True)
    sizes = (heads, kv_heads, dim, dim, width)
    want = TorchKernels(dtype).convolved_heads(x, *firsts, *sizes, batches["cpu"], cells["cpu"], eps=1e-5)
    close(kernels[dtype].convolved_heads(gpu(x), *firsts, *sizes, batches["cuda"], cells["cuda"], eps=1e-5), want, dtype)
    for name in ("keys", "values"):
        close(cells["cuda"].fields[name], cells["cpu"].fields[name], dtype)


def test_heads_that_do_not_fit_are_refused(kernels):
    from llmserve_amd.kernels.hip import KernelError

    sizes = (4, 1, 2, 16, 32, 32)
    x, firsts, taps, window, cells, batches = heads_case(torch.bfloat16, *sizes, [2, 3], [0, 4], 3, page=8)
    call = kernels[torch.bfloat16].convolved_heads
    rest = (4, 1, 16, 32, 32, batches["cuda"], cells["cuda"])
    good = dict(maps=2, taps=gpu(taps), window=gpu(window), eps=1e-5)
    call(gpu(x), *firsts, *rest, **good)
    for first, changed in ((firsts, {"taps": gpu(taps[:-1])}), (firsts, {"taps": gpu(taps.bfloat16())}), (firsts, {"window": None}), (firsts, {"window": gpu(window[:, 1:])}),
                           ((8, *firsts[1:]), {}), (firsts, {"q_weight": gpu(torch.ones(16))}), (firsts, {"maps": 3}), (firsts, {"temperature": (0.5, 0)})):
        with pytest.raises(KernelError):
            call(gpu(x), *first, *rest, **{**good, **changed})
    with pytest.raises(KernelError):  # pages of another head width
        call(gpu(x), *firsts, 4, 1, 16, 32, 64, batches["cuda"], cells["cuda"], **good)


# ---------------------------------------------------------------------------- attention

LONG = [([1, 1], [2500, 1300]), ([1], [4000]), ([2, 1], [1700, 2900])]  # few requests over long contexts: key splits


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,kv_heads,dim,vdim,page", [(4, 2, 64, 64, 16), (8, 1, 128, 128, 16), (6, 1, 48, 41, 8), (3, 3, 24, 20, 4), (40, 2, 32, 30, 16), (2, 1, 256, 252, 16)])
@pytest.mark.parametrize("counts,starts", STEPS + LONG)
@pytest.mark.parametrize("reach,gated,window", [(1, True, None), (9, False, None), (70, True, None), (300, True, None), (50, True, 77)])
def test_attention_with_a_bias_by_distance_and_a_gate(kernels, dtype, heads, kv_heads, dim, vdim, page, counts, starts, reach, gated, window):
    rows, layout, cells, batches = attention_case(dtype, heads, kv_heads, dim, page, counts, starts, window=window, row_stride=(heads + 2 * kv_heads) * dim + 24)
    table = 3.0 * torch.randn(heads, reach)
    gates = (2.0 * torch.randn(rows.shape[0], heads * vdim + 20)).to(dtype)
    plain, mine = TorchKernels(dtype), kernels[dtype]
    want = plain.paged_attention(rows, layout, batches["cpu"], cells["cpu"], 0.2, window, vdim=vdim, distance_bias=plain.prepare_distance_bias(table),
                                 gates=(gates, 12) if gated else None)
    got = mine.paged_attention(gpu(rows), layout, batches["cuda"], cells["cuda"], 0.2, window, vdim=vdim, distance_bias=mine.prepare_distance_bias(table),
                               gates=(gpu(gates), 12) if gated else None)
    close(got, want, dtype)


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_gate_without_a_bias(kernels, dtype):
    rows, layout, cells, batches = attention_case(dtype, 4, 2, 48, 16, [5, 1], [20, 70])
    gates = (2.0 * torch.randn(6, 4 * 45)).to(dtype)
    want = TorchKernels(dtype).paged_attention(rows, layout, batches["cpu"], cells["cpu"], 0.2, None, vdim=45, gates=(gates, 0))
    close(kernels[dtype].paged_attention(gpu(rows), layout, batches["cuda"], cells["cuda"], 0.2, None, vdim=45, gates=(gpu(gates), 0)), want, dtype)


@pytest.mark.parametrize("dtype", DTYPES)
def test_every_distance_has_its_own_bias(kernels, dtype):
    """A bias that towers over the scores at one distance: the query takes that key's value alone, wherever the key lies in
    its step, page and lane."""
    reach = 133
    rows, layout, cells, batches = attention_case(dtype, 2, 1, 32, 16, [150, 1, 1], [0, 200, 131])
    for distance in (0, 1, 2, 7, 8, 31, 32, 33, 100, 131, 132):
        table = torch.zeros(2, reach)
        table[:, distance] = 60.0
        plain, mine = TorchKernels(dtype), kernels[dtype]
        want = plain.paged_attention(rows, layout, batches["cpu"], cells["cpu"], 0.2, None, vdim=32, distance_bias=plain.prepare_distance_bias(table))
        got = mine.paged_attention(gpu(rows), layout, batches["cuda"], cells["cuda"], 0.2, None, vdim=32, distance_bias=mine.prepare_distance_bias(table))
        close(got, want, dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,kv_heads,width,vdim,page", [(4, 2, 64, 64, 16), (12, 2, 128, 128, 16), (6, 2, 96, 90, 8), (3, 3, 32, 7, 4), (40, 2, 32, 32, 16), (2, 1, 256, 250, 16), (1, 1, 160, 160, 16)])
@pytest.mark.parametrize("counts,starts", STEPS + LONG)
@pytest.mark.parametrize("factor", [0.7, -1.3])
def test_the_difference_of_two_maps(kernels, dtype, heads, kv_heads, width, vdim, page, counts, starts, factor):
    rows, layout, cells, batches = attention_case(dtype, heads, kv_heads, width, page, counts, starts, row_stride=(heads + 2 * kv_heads) * width + 16)
    for device, cell in cells.items():  # values are zeros beyond vdim, as the cache holds them
        cell.values[:, :, :, vdim:] = 0.0
    want = TorchKernels(dtype).difference_attention(rows, layout, batches["cpu"], cells["cpu"], 0.3, vdim, factor, 1e-5, 0.65)
    got = kernels[dtype].difference_attention(gpu(rows), layout, batches["cuda"], cells["cuda"], 0.3, vdim, factor, 1e-5, 0.65)
    assert got.shape == (sum(counts), heads * vdim)
    # (the norm stretches a small difference of two averages, and with it what bfloat16 weights of the values leave)
    close(got, want, dtype, **(dict(atol=4e-4, rtol=1e-3) if dtype == torch.float32 else dict(atol=6e-2, rtol=6e-2)))


@pytest.mark.parametrize("dtype", DTYPES)
def test_maps_do_not_mix(kernels, dtype):
    """Queries of one map alone: the other map's keys, whatever they are, give every key the same weight."""
    rows, layout, cells, batches = attention_case(dtype, 2, 1, 96, 16, [40, 1], [0, 90])
    view = rows[:, : 2 * 96].view(-1, 2, 96)
    view[:, :, 48:] = 0.0
    want = TorchKernels(dtype).difference_attention(rows, layout, batches["cpu"], cells["cpu"], 0.3, 96, 0.8, 1e-5, 0.65)
    cells["cuda"].keys[:, :, 6:] = 1.5  # pieces of the second map
    got = kernels[dtype].difference_attention(gpu(rows), layout, batches["cuda"], cells["cuda"], 0.3, 96, 0.8, 1e-5, 0.65)
    close(got, want, dtype, **(dict(atol=4e-4, rtol=1e-3) if dtype == torch.float32 else dict(atol=6e-2, rtol=6e-2)))


def test_finished_results_that_do_not_fit_are_refused(kernels):
    from llmserve_amd.kernels.hip import KernelError

    mine = kernels[torch.bfloat16]
    rows, layout, cells, batches = attention_case(torch.bfloat16, 4, 2, 64, 16, [1, 1], [5, 9])
    on = (gpu(rows), layout, batches["cuda"], cells["cuda"], 0.2)
    bias = mine.prepare_distance_bias(torch.zeros(4, 9))
    mine.paged_attention(*on, None, vdim=64, distance_bias=bias)
    for more in ({"vdim": 65}, {"vdim": -3}, {"distance_bias": mine.prepare_distance_bias(torch.zeros(3, 9))}, {"gates": (torch.zeros(2, 100, dtype=torch.bfloat16, device="cuda"), 0)},
                 {"soft_cap": 3.0}, {"chunk": 4}, {"gates": (torch.zeros(2, 256, device="cuda"), 0)}, {"out": torch.zeros(2, 100, dtype=torch.bfloat16, device="cuda")}):
        with pytest.raises(KernelError):
            mine.paged_attention(*on, None, **{"vdim": 64, "distance_bias": bias, **more})
    with pytest.raises(KernelError):
        mine.difference_attention(*on, 65, 0.5, 1e-5, 0.5)


# ---------------------------------------------------------------------------- experts beside another result


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("tokens,experts,top,hidden,size", [(3, 5, 2, 40, 24), (70, 9, 4, 320, 160), (33, 7, 1, 96, 33), (1, 4, 4, 1536, 64), (600, 5, 2, 192, 128), (400, 3, 3, 64, 320)])
@pytest.mark.parametrize("parts", [None, 1, 3])
def test_experts_with_a_limit_beside_another_result(kernels, dtype, tokens, experts, top, hidden, size, parts):
    torch.manual_seed(tokens + experts)
    plain, mine = TorchKernels(dtype), kernels[dtype]
    x = torch.randn(tokens, hidden).to(dtype)
    router = (3.0 * torch.randn(experts, hidden) / hidden**0.5).to(dtype)
    scores = plain.linear(x, plain.prepare_linear([router], None), out_dtype=torch.float32)
    want_chosen, want_weights = plain.route(scores, experts, None, top, 1.0, "softmax", renormalise=True)
    exact = torch.softmax(scores.gather(1, want_chosen.long()), dim=-1)
    torch.testing.assert_close(want_weights, exact, atol=1e-6, rtol=1e-5)  # a softmax over the chosen logits alone
    chosen, weights = mine.route(gpu(scores), experts, None, top, 1.0, "softmax", renormalise=True)
    assert torch.equal(chosen.cpu(), want_chosen)
    close(weights, exact, torch.float32)
    gates, ups = ([(torch.randn(size, hidden) / hidden**0.5).to(dtype) for _ in range(experts)] for _ in range(2))
    downs = [(torch.randn(hidden, size) / size**0.5).to(dtype) for _ in range(experts)]
    beside = None if parts is None else torch.randn(*((tokens, hidden) if parts == 1 else (parts, tokens, hidden)))
    want = plain.expert_feed_forward(x, plain.prepare_experts(ups, downs, "limited_swish", gates=gates, limit=0.9), want_chosen, want_weights, shared=beside)
    prepared = mine.prepare_experts([gpu(w) for w in ups], [gpu(w) for w in downs], "limited_swish", gates=[gpu(w) for w in gates], limit=0.9)
    got = mine.expert_feed_forward(gpu(x), prepared, chosen, weights, shared=None if beside is None else gpu(beside))
    close(got, want, dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("tokens", [1, 3, 8, 16, 17])
@pytest.mark.parametrize("experts,top,extra,hidden,groups,keep", [(5, 2, 0, 64, 1, 1), (16, 2, 0, 1536, 1, 1), (16, 4, 1, 352, 4, 2), (64, 8, 1, 96, 8, 3), (64, 16, 0, 96, 1, 1), (65, 3, 0, 64, 1, 1), (4, 4, 2, 40, 1, 1)])
@pytest.mark.parametrize("scoring,with_bias,with_correction,renormalise", [("softmax", False, False, True), ("sigmoid", True, True, False), ("softmax", True, True, True)])
def test_router_choice_and_sort_of_a_few_tokens(kernels, dtype, tokens, experts, top, extra, hidden, groups, keep, scoring, with_bias, with_correction, renormalise):
    """In one launch where the sizes allow it: scores, choices and weights as apart, and pairs sorted so that the experts'
    products find every token's rows."""
    torch.manual_seed(tokens * 100 + experts)
    plain, mine = TorchKernels(dtype), kernels[dtype]
    x = torch.randn(tokens, hidden).to(dtype)
    rows = [(3.0 * torch.randn(count, hidden) / hidden**0.5).to(dtype) for count in (experts, extra) if count]
    biases = [torch.randn(len(row)).to(dtype) for row in rows] if with_bias else None
    correction = 0.3 * torch.randn(experts) if with_correction else None
    size = 32
    gates, ups = ([(torch.randn(size, hidden) / hidden**0.5).to(dtype) for _ in range(experts)] for _ in range(2))
    downs = [(torch.randn(hidden, size) / size**0.5).to(dtype) for _ in range(experts)]
    options = (experts, None if correction is None else correction, top, 1.3, scoring, groups, keep, renormalise)
    prepared = plain.prepare_experts(ups, downs, "silu", gates=gates)
    scores, chosen, weights, _ = plain.route_product(x, plain.prepare_linear(rows, biases), prepared, *options)
    on = [gpu(w) for w in rows], [gpu(b) for b in biases] if with_bias else None
    there = mine.prepare_experts([gpu(w) for w in ups], [gpu(w) for w in downs], "silu", gates=[gpu(w) for w in gates])
    got_scores, got_chosen, got_weights, ordered = mine.route_product(
        gpu(x), mine.prepare_linear(*on), there, experts, None if correction is None else gpu(correction), *options[2:])
    assert (ordered is not None) == (dtype == torch.bfloat16 and tokens <= 16 and experts <= 64 and hidden % 32 == 0)
    torch.testing.assert_close(got_scores.cpu(), scores, atol=2e-4, rtol=2e-4)
    assert torch.equal(got_chosen.cpu(), chosen)
    torch.testing.assert_close(got_weights.cpu(), weights, atol=2e-4, rtol=2e-4)
    want = plain.expert_feed_forward(x, prepared, chosen, weights)
    close(mine.expert_feed_forward(gpu(x), there, got_chosen, got_weights, sorted_pairs=ordered), want, dtype)
