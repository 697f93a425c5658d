"""The kernels of the Dolezen parts, each alone against the same operation in elementary float32 torch (the CPU
stand-in of the kernel library), at sizes that are no powers of two and over steps that cut a request's tokens anywhere."""

from __future__ import annotations

import types

import pytest
import torch

from tests.test_gpu_sozavik_kernels import DTYPES, close, gpu, step_of
from tests.torch_kernels import TorchKernels

pytestmark = pytest.mark.gpu


@pytest.fixture(scope="module")
def kernels():
    from llmserve_amd.kernels import HipKernels

    return {dtype: HipKernels(dtype) for dtype in DTYPES}


def attention_case(dtype, heads, kv_heads, dim, page, counts, starts, window=None, chunk=None, row_stride=None):
    """(queries, keys and values; layout; cells and batches by device) of a step over cached keys.  The pages that a cache
    would have given back hold no number: a kernel that read one, even with a weight of zero, would show it."""
    from llmserve_amd.cache.cell import CacheCell
    from llmserve_amd.parts import HeadLayout, PagedKeyValue

    torch.manual_seed(dim + sum(counts) + (window or 0) + (chunk or 0))
    layout = HeadLayout(heads, kv_heads, dim, row_stride)
    need = PagedKeyValue(kv_heads, dim, window, 0, chunk)
    longest = max(s + c for s, c in zip(starts, counts))
    per = -(-longest // page)
    pages = per * len(counts) + 2
    fields = {name: (0.7 * torch.randn(pages, *shape)).to(dtype) for name, shape in need.page_fields(page).items()}
    for value in fields.values():
        value[pages - 1] = float("nan")  # the page that stands for every page given back
    tables = (torch.randperm(pages - 2) + 1)[: per * len(counts)].reshape(len(counts), per).to(torch.int32)
    slots = []
    for b, (start, count) in enumerate(zip(starts, counts)):
        tables[b, : need.first_read(start) // page] = pages - 1
        slots += [int(tables[b, p // page]) * page + p % page for p in range(start, start + count)]
    rows = (0.8 * torch.randn(sum(counts), layout.stride)).to(dtype)

    def batch_on(device):
        batch = step_of(counts, starts, list(range(len(counts))), device)
        batch.token_sequence = torch.cat([torch.full((c,), b) for b, c in enumerate(counts)]).to(torch.int32).to(device)
        batch.max_context_length = longest
        batch.context_lengths = torch.tensor([s + c for s, c in zip(starts, counts)], dtype=torch.int32).to(device)
        batch.groups = [types.SimpleNamespace(page_size=page, block_tables=tables.to(device), slot_mapping=torch.tensor(slots, dtype=torch.int32).to(device), width=per)]
        batch.padded_to = None
        return batch

    cells = {device: CacheCell(need, group=0, fields={name: value.clone().to(device) for name, value in fields.items()}) for device in ("cpu", "cuda")}
    return rows, layout, cells, {device: batch_on(device) for device in cells}


STEPS = [([1, 1, 1], [700, 3, 140]), ([33, 1, 7], [0, 90, 250]), ([300], [0]), ([64, 2, 17], [100, 511, 31]), ([1] * 9, [31, 32, 33, 63, 64, 0, 127, 128, 259])]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,kv_heads,dim,page", [(4, 2, 64, 16), (8, 1, 128, 16), (6, 1, 48, 8), (3, 3, 24, 4), (40, 2, 32, 16)])
@pytest.mark.parametrize("counts,starts", STEPS)
@pytest.mark.parametrize("chunk,with_sink", [(32, True), (50, False), (7, True), (128, True), (1, True), (None, True)])
def test_attention_in_chunks_with_a_sink(kernels, dtype, heads, kv_heads, dim, page, counts, starts, chunk, with_sink):
    """A query sees the keys of its own chunk alone, through every attention kernel, with key splits, in portions that cross
    chunks and in single tokens; rows with other columns behind the heads, results written into wider rows."""
    rows, layout, cells, batches = attention_case(dtype, heads, kv_heads, dim, page, counts, starts, chunk=chunk,
                                                  row_stride=(heads + 2 * kv_heads) * dim + 24)
    sinks = torch.randn(heads) + 1.0 if with_sink else None
    into = {device: torch.full((rows.shape[0], heads * dim + 40), 3.0, dtype=dtype, device=device) for device in cells}
    want = TorchKernels(dtype).paged_attention(rows, layout, batches["cpu"], cells["cpu"], 0.2, None, sinks=sinks, chunk=chunk, out=into["cpu"])
    assert not torch.isnan(want.float()).any()
    got = kernels[dtype].paged_attention(gpu(rows), layout, batches["cuda"], cells["cuda"], 0.2, None, sinks=gpu(sinks) if with_sink else None,
                                         chunk=chunk, out=into["cuda"])
    assert got.data_ptr() == into["cuda"].data_ptr()
    close(got, want, dtype)  # (the columns behind the result among them: untouched)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,kv_heads,dim,page", [(4, 2, 64, 16), (12, 2, 128, 16), (3, 3, 24, 4), (2, 1, 80, 8), (3, 1, 160, 16), (2, 1, 256, 16)])
@pytest.mark.parametrize("counts,starts", STEPS)
@pytest.mark.parametrize("chunk,window,with_sink", [(32, None, True), (50, None, False), (600, None, True), (1, None, True), (None, 33, False), (None, 600, True), (None, None, True)])
def test_store_and_attend_under_a_mask(kernels, dtype, heads, kv_heads, dim, page, counts, starts, chunk, window, with_sink):
    """The same with the step's keys and values stored first, by the attention's own kernel in a step of single tokens."""
    rows, layout, cells, batches = attention_case(dtype, heads, kv_heads, dim, page, counts, starts, window, chunk, (heads + 2 * kv_heads) * dim + 16)
    sinks = torch.randn(heads) + 1.0 if with_sink else None
    want = TorchKernels(dtype).rotate_store_attend(rows.clone(), layout, batches["cpu"], cells["cpu"], None, "none", 0.2, window, sinks=sinks, chunk=chunk)
    into = torch.full((rows.shape[0], heads * dim + 8), 3.0, dtype=dtype, device="cuda")
    got = kernels[dtype].rotate_store_attend(gpu(rows), layout, batches["cuda"], cells["cuda"], None, "none", 0.2, window,
                                             sinks=gpu(sinks) if with_sink else None, chunk=chunk, out=into)
    close(got[:, : heads * dim], want, dtype)
    assert torch.equal(got[:, heads * dim:].cpu(), torch.full((rows.shape[0], 8), 3.0, dtype=dtype))
    for name in ("keys", "values"):  # what was stored, where; every other entry as it was
        assert torch.equal(torch.nan_to_num(cells["cuda"].fields[name].cpu().float()), torch.nan_to_num(cells["cpu"].fields[name].float()))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("counts,starts", STEPS)
def test_attention_over_another_layers_keys(kernels, dtype, counts, starts):
    """Rows of queries alone, over pages that are only read, with a chunk shorter than the one the pages are kept for."""
    from llmserve_amd.parts import HeadLayout

    _, _, cells, batches = attention_case(dtype, 4, 2, 64, 16, counts, starts, chunk=96)
    for cell in cells.values():
        cell.writable = False
    layout = HeadLayout(6, 2, 64, 6 * 64)  # (more query heads a key head than its owner has)
    torch.manual_seed(3)
    rows, sinks = (0.8 * torch.randn(sum(counts), 6 * 64)).to(dtype), torch.randn(6)
    want = TorchKernels(dtype).paged_attention(rows, layout, batches["cpu"], cells["cpu"], 0.2, None, sinks=sinks, chunk=48)
    close(kernels[dtype].paged_attention(gpu(rows), layout, batches["cuda"], cells["cuda"], 0.2, None, sinks=gpu(sinks), chunk=48), want, dtype)


def test_masks_and_rows_that_do_not_fit_are_refused(kernels):
    from llmserve_amd.kernels.hip import KernelError

    library = kernels[torch.bfloat16]
    rows, layout, cells, batches = attention_case(torch.bfloat16, 4, 2, 64, 16, [1, 1], [5, 9], chunk=8)
    on = (gpu(rows), layout, batches["cuda"], cells["cuda"])
    with pytest.raises(KernelError):
        library.paged_attention(*on, 0.2, 16, chunk=8)  # a window and chunks
    with pytest.raises(KernelError):
        library.paged_attention(*on, 0.2, None, chunk=8, out=torch.empty((2, 4 * 64 - 8), dtype=torch.bfloat16, device="cuda"))
    with pytest.raises(KernelError):
        library.rotate_store_attend(*on, None, "none", 0.2, None, chunk=8, sinks=torch.zeros(3, device="cuda"))
    with pytest.raises(KernelError):
        library.paged_attention(gpu(rows[:, :-8].contiguous()), *on[1:], 0.2, None, chunk=8)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,width,dims", [(3, 8, 8), (2, 24, 10), (1, 64, 64), (5, 6, 2)])
def test_rotate_columns_in_half_pairs(kernels, dtype, heads, width, dims):
    torch.manual_seed(width)
    tokens, stride = 9, width + 5
    angles = torch.rand(tokens, dims // 2) * 6.0
    table = torch.stack([angles.cos(), angles.sin()], dim=-1).contiguous()
    x, out = torch.randn(tokens, 3 + heads * stride).to(dtype), torch.randn(tokens, 4 + heads * (width + 2)).to(dtype)
    for pairing in ("half", "adjacent"):
        want = TorchKernels(dtype).rotate_columns(x, 3, stride, heads, width, table, dims, out.clone(), 4, width + 2, pairing=pairing)
        close(kernels[dtype].rotate_columns(gpu(x), 3, stride, heads, width, gpu(table), dims, gpu(out), 4, width + 2, pairing=pairing), want, dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows", [1, 5, 8, 16, 17, 40, 64, 100, 300])
@pytest.mark.parametrize("inner,outputs,first", [(64, 96, 0), (64, 100, 37), (40, 27, 3), (256, 512, 128), (1536, 2048, 512), (1024, 70, 6)])
def test_a_product_with_an_activated_tail(kernels, dtype, rows, inner, outputs, first):
    """Every product kernel for a few rows with the activation in its epilogue, and the kernel behind the others; whole
    results and results beside other columns."""
    torch.manual_seed(rows + outputs)
    x = torch.randn(rows, inner).to(dtype)
    weight, bias = (torch.randn(outputs, inner) / inner ** 0.5).to(dtype), (0.5 * torch.randn(outputs)).to(dtype)
    plain, library = TorchKernels(dtype), kernels[dtype]
    more = {"atol": 4e-2, "rtol": 3e-2} if dtype == torch.bfloat16 else {"atol": 1e-4, "rtol": 1e-4}
    for biases in (None, [bias]):
        prepared = library.prepare_linear([gpu(weight)], [gpu(b) for b in biases] if biases else None)
        for activation in ("squared_relu", "relu"):
            want_rows, want = plain.activated_linear(x, plain.prepare_linear([weight], biases), activation, first)
            got_rows, got = library.activated_linear(gpu(x), prepared, activation, first)
            close(got, want, dtype, **more)
            if first:
                close(got_rows[:, :first], want_rows[:, :first], dtype, **more)
            into = torch.full((rows, 16 + outputs - first + 8), 3.0, dtype=dtype, device="cuda")
            _, got = library.activated_linear(gpu(x), prepared, activation, first, out=into, out_first=16)
            close(got[:, 16 : 16 + outputs - first], want, dtype, **more)
            assert (got[:, :16] == 3.0).all() and (got[:, 16 + outputs - first:] == 3.0).all()
    from llmserve_amd.kernels.hip import KernelError

    for wrong in (dict(activation="limited_swish"), dict(activation="cube"), dict(activation="relu", first=outputs),
                  dict(activation="relu", out=torch.empty((rows, outputs - 1), dtype=dtype, device="cuda"))):
        with pytest.raises(KernelError):
            library.activated_linear(gpu(x), prepared, **wrong)


@pytest.mark.parametrize("dtype", DTYPES)
def test_squared_relu_elementwise_in_gates_and_in_experts(kernels, dtype):
    torch.manual_seed(1)
    plain, library = TorchKernels(dtype), kernels[dtype]
    x = torch.randn(7, 40).to(dtype)
    close(library.activate(gpu(x), "squared_relu"), plain.activate(x, "squared_relu"), dtype)
    gate, up = ((torch.randn(24, 40) / 6).to(dtype) for _ in range(2))
    want = plain.gated_linear(x, plain.prepare_gated_linear(gate, up, "squared_relu"))
    close(library.gated_linear(gpu(x), library.prepare_gated_linear(gpu(gate), gpu(up), "squared_relu")), want, dtype, atol=4e-2, rtol=3e-2)
    ups, downs = [(torch.randn(24, 40) / 6).to(dtype) for _ in range(3)], [(torch.randn(40, 24) / 5).to(dtype) for _ in range(3)]
    chosen, weights = torch.tensor([[0], [2], [1], [1], [0], [2], [2]], dtype=torch.int32), torch.rand(7, 1)
    want = plain.expert_feed_forward(x, plain.prepare_experts(ups, downs, "squared_relu"), chosen, weights)
    prepared = library.prepare_experts([gpu(w) for w in ups], [gpu(w) for w in downs], "squared_relu")
    close(library.expert_feed_forward(gpu(x), prepared, gpu(chosen), gpu(weights)), want, dtype, **({"atol": 5e-2, "rtol": 5e-2} if dtype == torch.bfloat16 else {}))


@pytest.mark.parametrize("dtype", DTYPES)
def test_scaled_embedding(kernels, dtype):
    torch.manual_seed(2)
    table, ids = torch.randn(31, 70).to(dtype), torch.tensor([3, 30, 0, 3], dtype=torch.int32)
    for scale in (1.0, 16.0, 0.37):
        close(kernels[dtype].embedding(gpu(table), gpu(ids), scale), TorchKernels(dtype).embedding(table, ids, scale), torch.float32)


@pytest.mark.parametrize("rows", [300, 600])
@pytest.mark.parametrize("with_bias", [False, True])
def test_products_over_slices_of_a_long_k(kernels, rows, with_bias):
    """The library's product cut over K into partial sums, with a bias (counted once) and without."""
    torch.manual_seed(rows)
    inner, outputs = 16384, 128
    library = kernels[torch.bfloat16]
    assert library._library_splits(rows, outputs, inner) > 1
    x, weight = torch.randn(rows, inner).to(torch.bfloat16), (torch.randn(outputs, inner) / inner ** 0.5).to(torch.bfloat16)
    bias = torch.randn(outputs).to(torch.bfloat16)
    want = x.float() @ weight.float().T + (bias.float() if with_bias else 0.0)
    prepared = library.prepare_linear([gpu(weight)], [gpu(bias)] if with_bias else None)
    for _ in range(2):
        got = library.linear(gpu(x), prepared, out_dtype=torch.float32, partial=True)
        assert got.ndim == 3
        close(got.sum(0), want, torch.float32, atol=2e-3, rtol=1e-3)
