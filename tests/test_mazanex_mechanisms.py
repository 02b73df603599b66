"""Each mechanism of Mazanex alone, against the plain implementation's function for it: the kernel
set's operation on the engine's own layouts (pages, block tables, state slots), once as the PyTorch
reference on the CPU and once as the HIP kernel on the GPU.  Where random numbers would hide a
fault, one query and key are scaled so that one score stands out."""
import math

import pytest
import torch

import helpers as H          # noqa: F401
import plain_mazanex as P
from test_vivevik_mechanisms import BACKENDS, DTYPES, F64, Paged, close, ops_of, randn
from llm_inference_lab_amd.cache.layout import value_quads
from llm_inference_lab_amd.parts.base import PendingSums
from llm_inference_lab_amd.parts.positions import RotaryEmbedding


def ints(values, dev):
    return torch.tensor(values, dtype=torch.int32, device=dev)


def batch(spans, dev):
    """``spans``: rows each request of a step brings -> (q_start, row_req) on the device."""
    starts = [0]
    for n in spans:
        starts.append(starts[-1] + n)
    return ints(starts, dev), ints([b for b, n in enumerate(spans) for _ in range(n)], dev)


# ------------------------------------------------------------------ the stream
@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("width", [7, 8, 72, 1000, 2600])
def test_token_shift_over_portions_and_slots(backend, width):
    """Three requests over two steps (portions, single rows) with slots in scattered places: every row
    mixed with the one before it in its own sequence, zeros before the first; several mixes at once;
    float32 rows to both dtypes, bfloat16 rows to bfloat16."""
    ops = ops_of(backend)
    dev = ops.device
    lengths, first = [9, 2, 5], [4, 1, 3]
    mix = torch.rand(3, width, generator=torch.Generator().manual_seed(1))
    for src, dst in ((torch.float32, torch.float32), (torch.float32, torch.bfloat16), (torch.bfloat16, torch.bfloat16)):
        h = [randn(n, width, seed=10 + b, scale=2.0).to(src) for b, n in enumerate(lengths)]
        state = torch.zeros(6, width, dtype=src, device=dev)
        state[1] = 7.0                               # (a slot nobody uses stays as it is)
        slots = ints([4, 0, 5], dev)
        for spans in ([(0, f) for f in first], [(f, n) for f, n in zip(first, lengths)]):
            rows = torch.cat([h[b][lo:hi] for b, (lo, hi) in enumerate(spans)]).to(dev)
            q_start, row_req = batch([hi - lo for lo, hi in spans], dev)
            out = torch.full((3, rows.shape[0], width), float("nan"), dtype=dst, device=dev)
            ops.shift_mix(rows, mix.to(dev), state, row_req, q_start, slots, out)
            for m in range(3):
                want = torch.cat([P.token_shift(h[b].to(F64), mix[m].to(F64))[lo:hi] for b, (lo, hi) in enumerate(spans)])
                close(out[m], want, dst, f"mix {m}", f32=1e-6, bf16=8e-3)
        for b, slot in enumerate((4, 0, 5)):
            assert torch.equal(state[slot].cpu(), h[b][-1])
        assert float((state[1].float() - 7.0).abs().max()) == 0.0


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("hidden", [8, 72, 1000, 2600])
def test_sums_into_the_stream_and_what_comes_out_of_their_launch(backend, hidden):
    """The norm of a result on its way into the stream, with a rounded copy, and, for rows that are
    requests of their own, with the next run's token shift; the result whole or in pieces."""
    ops = ops_of(backend)
    dev = ops.device
    n = 5
    w = (1.0 + randn(hidden, seed=2, scale=0.3)).to(dev)
    pieces = randn(3, n, hidden, seed=4).to(dev)
    for y, y64 in ((pieces[0].clone(), pieces[0].cpu().to(F64)), (PendingSums(pieces, 3), pieces.cpu().to(F64).sum(0))):
        for dtype in DTYPES:
            x = randn(n, hidden, seed=3).to(dev)
            want = x.cpu().to(F64) + P.rms_norm(y64, w.cpu().to(F64), 1e-4)
            copy = torch.full((n, hidden), float("nan"), dtype=dtype, device=dev)
            ops.rmsnorm_add(y, w, 1e-4, x, copy=copy)
            close(x, want, torch.float32, "stream += norm(y)", f32=3e-6)
            close(copy, want, dtype, "its copy", f32=3e-6)
            x = randn(n, hidden, seed=3).to(dev)
            mix = torch.rand(1, hidden, generator=torch.Generator().manual_seed(6)).to(dev)
            state = randn(7, hidden, seed=7).to(dev)
            before = state.cpu().to(F64)
            slots = [6, 2, 0, 5, 3]
            out = torch.full((1, n, hidden), float("nan"), dtype=dtype, device=dev)
            ops.rmsnorm_add(y, w, 1e-4, x, shift=(mix, state, ints(slots, dev), out))
            close(x, want, torch.float32, "stream += norm(y), with the shift", f32=3e-6)
            close(out[0], want + (before[slots] - want) * mix.cpu().to(F64), dtype, "the shifted rows", f32=3e-6)
            close(state[slots], want, torch.float32, "the slots take the new rows", f32=3e-6)
            assert torch.equal(state[[1, 4]].cpu().to(F64), before[[1, 4]])


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("hidden", [8, 72, 1000, 2600])
def test_half_the_sum_of_two_normed_results(backend, hidden):
    ops = ops_of(backend)
    dev = ops.device
    y1, y2 = randn(6, hidden, seed=1, scale=40.0).to(dev), randn(6, hidden, seed=2, scale=0.02).to(dev)
    w1, w2 = ((1.0 + randn(hidden, seed=s, scale=0.3)).to(dev) for s in (3, 4))
    s64 = 0.5 * (P.rms_norm(y1.cpu().to(F64), w1.cpu().to(F64), 1e-5) + P.rms_norm(y2.cpu().to(F64), w2.cpu().to(F64), 1e-5))
    out = torch.full((6, hidden), float("nan"), device=dev)
    ops.normed_sum(out, y1, w1, 0.5, y2, w2, 0.5, 1e-5)
    close(out, s64, torch.float32, "the sum", f32=3e-6)
    wa = (1.0 + randn(hidden, seed=5, scale=0.3)).to(dev)
    for dtype in (None,) + tuple(DTYPES):
        x = randn(6, hidden, seed=6).to(dev)
        want = x.cpu().to(F64) + P.rms_norm(s64, wa.cpu().to(F64), 1e-3)
        copy = None if dtype is None else torch.full((6, hidden), float("nan"), dtype=dtype, device=dev)
        ops.normed_sum(x, y1, w1, 0.5, y2, w2, 0.5, 1e-5, add=(wa, 1e-3), copy=copy)
        close(x, want, torch.float32, "its norm into the stream", f32=5e-6)
        if copy is not None:
            close(copy, want, dtype, "the copy", f32=5e-6)


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows,count,columns", [(3, 5, 8), (300, 52, 56), (9, 1000, 1000), (2, 19000, 19000), (300, 4864, 4864),
                                                (2, 30000, 30000)])
def test_normed_powers(backend, dtype, rows, count, columns):
    """``a N(z) + b N(z^2) + c N(z^3) + e`` over rows with padding behind them, from a row in one thread's
    registers to rows that are read twice."""
    if backend == "emu" and rows * columns > 100000:
        pytest.skip("the references on the CPU take the small shapes; the kernels all of them")
    ops = ops_of(backend)
    z = randn(rows, columns, seed=1, scale=1.7)
    z[:, count:] = 0.0
    coef = torch.tensor([0.8, -0.6, 0.3, 0.25])
    out = torch.full((rows, columns), float("nan"), dtype=dtype, device=ops.device)
    ops.poly_norm(z.to(ops.device), coef.to(ops.device), 1e-4, count, out)
    close(out[:, :count], P.poly_norm(z[:, :count].to(F64), *coef.to(F64), 1e-4), dtype, "normed powers", f32=5e-6)
    assert torch.isfinite(out.float()).all()       # (the padding meets zero columns of the next product)


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows", [1, 9, 40, 64, 130])
def test_products_with_inputs_of_their_own(backend, dtype, rows):
    """Five matrices of unequal heights, each with its own rows: one launch at few rows (heights that
    are no multiples of 16 included), a product each at many."""
    ops = ops_of(backend)
    dev = ops.device
    heights, k = [24, 40, 16, 72, 5], 96
    x = randn(5, rows, k, seed=1).to(dtype).to(dev)
    ws = [randn(n, k, seed=2 + i, scale=0.3).to(dtype) for i, n in enumerate(heights)]
    offsets, at = [], 0
    for n in heights:
        offsets.append(at)
        at += (n + 15) // 16 * 16
    out = torch.zeros(rows, at, device=dev)
    ops.segmented_products(x, ops.prepare_segments([w.to(dev) for w in ws]), out, offsets)
    for i, (w, n) in enumerate(zip(ws, heights)):
        close(out[:, offsets[i]:offsets[i] + n], x[i].cpu().to(F64) @ w.to(F64).T, torch.float32, f"segment {i}", f32=2e-5)


# ------------------------------------------------------------------ projections on their way to the pages
@pytest.mark.parametrize("dim,dims,base", [(32, 32, 1e4), (20, 8, 50.0), (10, 2, 7.0)])
def test_frequencies_of_halves(dim, dims, base):
    part = RotaryEmbedding(dim=dim, theta=base, rotary_dim=dims)
    part.bind({}, ops_of("emu"), torch.float32)
    freq, turning = part.half_table()
    assert turning == dims
    assert torch.allclose(freq.to(F64), torch.tensor([base ** (-2.0 * i / dims) for i in range(dims // 2)], dtype=F64),
                          rtol=1e-6, atol=0)


def shaped(u, w, positions, heads, D, rot, eps):
    """Convolution, rotation and unit norm of one projection's channels (plain)."""
    x = P.short_conv(u, w).view(u.shape[0], heads, D)
    if rot:
        x = P.rotate_halves(x, positions, rot)
    return P.unit_rms(x, eps)


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H_,G,D,E,taps,dims", [(3, 1, 16, 24, 4, 16), (4, 2, 24, 8, 3, 6), (6, 3, 9, 16, 2, 4), (2, 2, 32, 40, 1, 0),
                                                (5, 1, 14, 12, 7, 14), (70, 2, 192, 96, 4, 128)])
@pytest.mark.parametrize("plan", ["short", "long"])
def test_bias_convolution_rotation_unit_norm_and_the_cache_write(backend, dtype, H_, G, D, E, taps, dims, plan):
    """Requests in portions (down to one row) and then single rows, against whole sequences, with few
    rows in a step and with many (short ones between long ones, and a description with room for more
    requests than the step has, which says something stale there): biases
    enter the convolution's inputs (but not what stands before a sequence), the last inputs are
    carried in slots, the first ``dims`` channels of a head turn in halves, the norm comes last."""
    if backend == "emu" and H_ > 10:
        pytest.skip("the references on the CPU take the small shapes; the kernels all of them")
    ops = ops_of(backend)
    dev = ops.device
    laid = (D + 31) // 32 * 32
    portions = {"short": ([17, 1], [2, 3], [5, 16], [1, 1], [1, 1], [15, 1]),
                "long": ([66, 1, 2], [2, 67, 1], [1, 2, 70], [1, 1, 1], [64, 1, 3])}[plan]
    lengths = [sum(spans[b] for spans in portions) for b in range(len(portions[0]))]
    stale = [-1, 5, 10 ** 6, 0] if plan == "long" else []
    slots = ints([3, 1, 4][:len(lengths)] + [2] * len(stale), dev)
    rot = dict(dims=dims, base=60.0) if dims else None
    sizes = (H_ * D, G * D, G * E)
    total = sum(sizes)
    ld = total + 11
    proj = [randn(n, ld, seed=5 + b, scale=2.0) for b, n in enumerate(lengths)]
    bias = randn(total, seed=8)
    conv = randn(total, taps, seed=9, scale=0.6)
    cache = Paged(ops, dtype, lengths, G, laid, E)
    state = torch.zeros(5, taps - 1, total, device=dev) if taps > 1 else None
    freq = None
    if dims:
        freq = torch.tensor([60.0 ** (-2.0 * i / dims) for i in range(dims // 2)], dtype=F64).float().to(dev)
    want_q, want_k, want_v = [], [], []
    for b, n in enumerate(lengths):
        u, w = proj[b][:, :total].to(F64) + bias.to(F64), conv.to(F64)
        cut = [0, sizes[0], sizes[0] + sizes[1], total]
        want_q.append(shaped(u[:, :cut[1]], w[:cut[1]], range(n), H_, D, rot, 1e-4))
        want_k.append(shaped(u[:, cut[1]:cut[2]], w[cut[1]:cut[2]], range(n), G, D, rot, 1e-4))
        want_v.append(P.short_conv(u[:, cut[2]:], w[cut[2]:]).view(n, G, E))
    done = [0] * len(lengths)
    for spans in portions:
        rows = torch.cat([proj[b][done[b]:done[b] + n] for b, n in enumerate(spans)]).to(dev)
        positions = [done[b] + i for b, n in enumerate(spans) for i in range(n)]
        q_start, row_req = batch(spans, dev)
        q = torch.full((rows.shape[0], H_ * laid), float("nan"), dtype=dtype, device=dev)
        ops.project_conv_write(rows, H_, G, D, E, bias.to(dev), conv.t().contiguous().to(dev), state,
                               torch.cat([q_start, ints(stale, dev)]), slots, freq, dims, "halves", 1e-4, q, cache.k_cache,
                               cache.v_cache, cache.page, ints(positions, dev), row_req, cache.table,
                               all(n == 1 for n in spans))
        got = q.view(rows.shape[0], H_, laid)
        want = torch.cat([want_q[b][done[b]:done[b] + n] for b, n in enumerate(spans)])
        close(got[..., :D], want, dtype, f"queries of {spans}", f32=2e-5)
        assert float(got[..., D:].float().abs().max() if laid > D else 0.0) == 0.0
        done = [d + n for d, n in zip(done, spans)]
    assert done == lengths
    for b, n in enumerate(lengths):
        for pos in range(n):
            page = int(cache.table[b, pos // 16])
            close(cache.k_cache[page, :, pos % 16, :D], want_k[b][pos], dtype, f"key {pos} of request {b}", f32=2e-5)
            close(value_quads(cache.v_cache[page])[:, (pos % 16) >> 2, :, pos & 3], want_v[b][pos], dtype,
                  f"value {pos} of request {b}", f32=1e-5)


@pytest.mark.parametrize("backend", BACKENDS)
def test_neighbouring_channels_turn_in_the_same_kernel(backend):
    """The other pairing, without a convolution, a bias or a norm."""
    import plain_ninisun
    ops = ops_of(backend)
    dev = ops.device
    n, H_, G, D, E = 9, 2, 1, 32, 16
    proj = randn(n, (H_ + G) * D + G * E, seed=1)
    cache = Paged(ops, torch.float32, [n], G, D, E)
    rot = dict(dims=12, base=30.0)
    freq, _ = plain_ninisun.rotary_frequencies(rot)
    q = torch.empty(n, H_ * D, device=dev)
    q_start, row_req = batch([n], dev)
    ops.project_conv_write(proj.to(dev), H_, G, D, E, None, None, None, q_start, ints([0], dev), freq.float().to(dev), 12,
                           "neighbours", None, q, cache.k_cache, cache.v_cache, cache.page, ints(list(range(n)), dev), row_req,
                           cache.table, False)
    want = plain_ninisun.rotate_pairs(proj[:, :H_ * D].to(F64).view(n, H_, D), range(n), rot)
    close(q, want.reshape(n, -1), torch.float32, "queries", f32=1e-5)


# ------------------------------------------------------------------ attention over chunks
SHAPES = [(4, 2, 16, 24), (4, 2, 32, 16), (8, 2, 64, 64), (3, 1, 64, 48), (6, 3, 96, 32), (4, 1, 128, 128), (2, 2, 32, 208)]


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H_,G,D,E", SHAPES)
@pytest.mark.parametrize("chunk", [1, 7, 16, 37, 64, 1000, None])
def test_chunks_sinks_and_gates_per_channel(backend, dtype, H_, G, D, E, chunk):
    """Portions behind a history, tiles of rows that hold two requests or cross a chunk's edge, decoded
    rows; queries made to point at the first key of their chunk (seen), the last key of the chunk
    before (not seen) and far keys; sinks of the scores' size; outputs gated channel by channel."""
    if backend == "emu" and (H_ * (D + E) > 600 or chunk in (16, 1000)):
        pytest.skip("the references on the CPU take the small shapes; the kernels all of them")
    ops = ops_of(backend)
    dev = ops.device
    lengths, new = [150, 45, 75, 1], [70, 45, 1, 1]
    c = chunk or 10 ** 6
    ks = [randn(n, G, D, seed=30 + i) for i, n in enumerate(lengths)]
    vs = [randn(n, G, E, seed=40 + i) for i, n in enumerate(lengths)]
    qs = [randn(n, H_, D, seed=50 + i) for i, n in enumerate(lengths)]
    for b, n in enumerate(lengths):
        for i in range(n - new[b], n):
            edge = i // c * c
            target = (edge, edge - 1, max(edge, i - 40), i)[i % 4]         # first of the chunk, just outside, far, itself
            if 0 <= target:
                for h in range(H_):
                    key = ks[b][target, h // (H_ // G)]
                    qs[b][i, h] = key * 6.0 / key.norm()
    cache = Paged(ops, dtype, lengths, G, D, E, seed=3)
    for b, n in enumerate(lengths):
        cache.write(torch.cat([torch.zeros(n, H_ * D), ks[b].reshape(n, -1), vs[b].reshape(n, -1)], 1), H_, list(range(n)),
                    [b] * n)
    rows_q = torch.cat([qs[b][n - new[b]:] for b, n in enumerate(lengths)]).to(dtype)
    positions = [p for b, n in enumerate(lengths) for p in range(n - new[b], n)]
    row_req = [b for b in range(len(lengths)) for _ in range(new[b])]
    sink = torch.tensor([1.5 * h - 1.0 for h in range(H_)])
    gate = randn(len(positions), 5 + H_ * E, seed=60, scale=2.0)
    scale = 0.8 / math.sqrt(D) * 4.0
    pick = getattr(ops, "windowed_attention_long_rows", None)
    long_from = pick(dtype, D, E, cache.page) if pick is not None else 0
    q_start, _ = batch(new, dev)
    launches = (1 if any(n < long_from for n in new) else 0) | (2 if any(n >= long_from for n in new) else 0)
    for gated in (False, True):
        out = torch.full((len(positions), H_ * E), float("nan"), dtype=dtype, device=dev)
        ops.sink_window_attention(rows_q.reshape(len(positions), -1).to(dev), H_, G, D, E, cache.k_cache, cache.v_cache,
                                  cache.table, cache.page, ints(positions, dev), ints(row_req, dev), None, 0, sink.to(dev), scale,
                                  out, q_start, long_from, launches if long_from else 1, min(150, c),
                                  chunk=chunk, gate=(gate.to(dev), 5) if gated else None)
        at = 0
        for b, n in enumerate(lengths):
            want = P.chunked_sink_attention(rows_q[at:at + new[b]].to(F64), ks[b].to(dtype).to(F64), vs[b].to(dtype).to(F64),
                                            scale, chunk, sink.to(F64)).reshape(new[b], -1)
            if gated:
                want = want * torch.sigmoid(gate[at:at + new[b], 5:].to(F64))
            close(out[at:at + new[b]], want, dtype, f"request {b}, gated {gated}", f32=3e-5, bf16=2.5e-2)
            at += new[b]


@pytest.mark.parametrize("size", [1, 2, 5, 16, 33])
def test_the_oracle_s_chunks(size):
    for i in range(70):
        seen = [j for j in range(70) if P.visible(i, j, size)]
        assert seen == list(range(i // size * size, i + 1))


# ------------------------------------------------------------------ recurrences
@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("rank", [3, 16, 64])
def test_decays_and_their_logarithms(backend, rank):
    ops = ops_of(backend)
    dev = ops.device
    rows, channels = 7, 39
    low = randn(rows, rank + 5, seed=1, scale=2.0).to(dev)
    w2, bias = randn(channels, rank, seed=2, scale=0.7).to(dev), randn(channels, seed=3, scale=2.0).to(dev)
    z = lambda x: x @ w2.cpu().to(F64).T + bias.cpu().to(F64)
    low64 = low.cpu().to(F64)[:, :rank]
    for kind, tau, want in (("double_exp", 1.0, torch.exp(-torch.exp(z(torch.tanh(low64))))),
                            ("sigmoid", 7.0, torch.sigmoid(z(low64)) ** (1 / 7.0))):
        out = torch.full((rows, channels), float("nan"), device=dev)
        ops.gla_decay(low, rank, w2, bias, tau, out, kind)
        close(out, want, torch.float32, kind, f32=5e-6)
        ops.gla_decay(low, rank, w2, bias, tau, out, kind, as_log=True)
        close(out, torch.clamp(torch.log2(want), min=-60.0), torch.float32, kind + ", log2", f32=2e-5)


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("cap", [1.5, 15.0])
def test_gates_of_a_matrix_memory(backend, cap):
    """Gates and running maxima of two requests over several steps (one longer than a block's tile), from
    the maxima in their slots; the very first from 0, not from minus infinity."""
    ops = ops_of(backend)
    dev = ops.device
    heads, lengths = 3, [1400, 6] if backend == "hip" else [140, 6]
    proj = [randn(n, 2 * heads + 4, seed=1 + b, scale=6.0) for b, n in enumerate(lengths)]
    proj[0][:40, 1:1 + heads] -= 30.0                  # (small input gates: the maximum decays from 0)
    bi, bf = randn(heads, seed=5).to(dev), randn(heads, seed=6, scale=2.0).to(dev)
    slots, maxima_state = ints([2, 0], dev), torch.zeros(3, heads, device=dev)
    want = []
    for b, n in enumerate(lengths):
        x = proj[b].to(F64)
        i = cap * torch.tanh((x[:, 1:1 + heads] + bi.cpu()) / cap)
        f = torch.nn.functional.logsigmoid(cap * torch.tanh((x[:, 1 + heads:1 + 2 * heads] + bf.cpu()) / cap))
        m, rows = torch.zeros(heads, dtype=F64), []
        for t in range(n):
            new = torch.maximum(f[t] + m, i[t])
            rows.append((f[t] + m - new, i[t] - new, new))
            m = new
        want.append([torch.stack(v) for v in zip(*rows)])
    done = [0, 0]
    for spans, as_log in (([3, 1], False), ([lengths[0] - 4, 4], True), ([1, 1], False)):
        rows = torch.cat([proj[b][done[b]:done[b] + n] for b, n in enumerate(spans)]).to(dev)
        q_start, _ = batch(spans, dev)
        keep, take, maxima = (torch.full((rows.shape[0], heads), float("nan"), device=dev) for _ in range(3))
        ops.memory_gates(rows, 1, 1 + heads, bi, bf, cap, heads, maxima_state, q_start, slots, 2, keep, take, maxima, as_log=as_log)
        part = [torch.cat([want[b][i][done[b]:done[b] + n] for b, n in enumerate(spans)]) for i in range(3)]
        kept = torch.clamp(part[0] / math.log(2.0), min=-60.0) if as_log else torch.exp(part[0])
        close(keep, kept, torch.float32, "keep", f32=3e-5)
        close(take, torch.exp(part[1]), torch.float32, "take", f32=3e-5)
        close(maxima, part[2], torch.float32, "maxima", f32=1e-5)
        done = [d + n for d, n in zip(done, spans)]
    assert done == lengths


class Recurrence:
    """Three requests with projections, decays or gates, and the plain recurrence over the whole of each."""

    def __init__(self, kind, heads, D, E, lengths, seed, harsh=False):
        self.kind, self.heads, self.D, self.E, self.lengths = kind, heads, D, E, lengths
        hd, he = heads * D, heads * E
        self.off = (3, 3 + hd, 3 + 2 * hd, 3 + 2 * hd + he)
        self.ld = 3 + 2 * hd + 2 * he + 6
        self.q_scale, self.eps = 0.7, 1e-4
        self.gate = "sigmoid" if kind == "memory" else "silu"
        self.weight = 1.0 + randn(he if kind != "decay" else E, seed=seed + 1, scale=0.3)
        self.bonus = randn(hd, seed=seed + 2) if kind == "bonus" else None
        self.proj = [randn(n, self.ld, seed=seed + 10 + b) for b, n in enumerate(lengths)]
        self.logs, self.take, self.maxima, self.want, self.last = [], [], [], [], []
        for b, n in enumerate(lengths):
            g = torch.Generator().manual_seed(seed + 20 + b)
            width = hd if kind != "memory" else heads
            # (harsh: some channels forget everything at a row, others nothing)
            log = -torch.exp(3.5 * torch.randn(n, width, generator=g) - 1.0) if harsh else -torch.rand(n, width, generator=g)
            p = self.proj[b].to(F64)
            q, k = (p[:, o:o + hd].view(n, heads, D) for o in self.off[:2])
            v = p[:, self.off[2]:self.off[2] + he].view(n, heads, E)
            q = q * self.q_scale
            if kind == "decay":
                o, last = P.decay_rule(q, k, v, torch.exp(log.to(F64)).view(n, heads, D))
            elif kind == "bonus":
                o, last = P.bonus_rule(q, k, v, torch.exp(log.to(F64)).view(n, heads, D), self.bonus.to(F64).view(heads, D))
            else:
                # log gates (f = log, i) -> what the kernels are given
                i = 2.0 * torch.randn(n, heads, generator=g)
                o, last = P.matrix_memory(q, k, v, i.to(F64), log.to(F64))
                m, keep, take, maxima = torch.zeros(heads, dtype=F64), [], [], []
                for t in range(n):
                    new = torch.maximum(log[t].to(F64) + m, i[t].to(F64))
                    keep.append(log[t].to(F64) + m - new)
                    take.append(torch.exp(i[t].to(F64) - new))
                    maxima.append(new)
                    m = new
                log = torch.stack(keep).float()
                self.take.append(torch.stack(take).float())
                self.maxima.append(torch.stack(maxima).float())
            gate = p[:, self.off[3]:self.off[3] + he]
            gate = P.silu(gate) if self.gate == "silu" else torch.sigmoid(gate)
            w = self.weight.to(F64).repeat(heads) if kind == "decay" else self.weight.to(F64)
            self.logs.append(log)
            self.want.append(P.unit_rms(o, self.eps).reshape(n, he) * w * gate)
            self.last.append(last)

    def step(self, ops, spans, slots, state, norm_state, how, dtype):
        """One call over ``spans = [(first, end)]``: ``how`` is "scan", "chunks" or an int (the scan in chunks)."""
        dev = ops.device
        cat = lambda xs: torch.cat([xs[b][lo:hi] for b, (lo, hi) in enumerate(spans)]).to(dev)
        proj, logs = cat(self.proj), cat(self.logs)
        q_start, _ = batch([hi - lo for lo, hi in spans], dev)
        rows, n = proj.shape[0], len(spans)
        heads, D, E = self.heads, self.D, self.E
        out = torch.full((rows, heads * E), float("nan"), dtype=dtype, device=dev)
        take, maxima = (cat(self.take), cat(self.maxima)) if self.kind == "memory" else (None, None)
        nan = lambda *shape: torch.full(shape, float("nan"), device=dev)
        weight, bonus = self.weight.to(dev), None if self.bonus is None else self.bonus.to(dev)
        if how == "chunks":
            most = rows // 64 + n
            kind = {} if bonus is None else dict(bonus=bonus)
            if self.kind == "memory":
                kind["memory"] = (take, norm_state, maxima, nan(most, heads, D))
            ops.chunk_scan(proj, *self.off, self.q_scale, heads, D, E, torch.clamp(logs / math.log(2.0), min=-60.0), state, q_start,
                           slots, n, nan(most, heads, D, E), nan(most, heads, D), weight, self.eps, self.gate, 0, out, **kind)
            return out
        chunk = 0 if how == "scan" else how
        most = rows // chunk + n if chunk else 0
        parts = nan(rows, heads, ops.gla_slices(D), E)
        kind, norm, decay = {}, {}, torch.exp(logs)
        if bonus is not None:
            kind["bonus"] = bonus
        if self.kind == "memory":
            norm = dict(norm_parts=nan(rows, heads, ops.gla_slices(D)), maxima=maxima)
            kind["memory"] = (decay, take, norm_state, norm["norm_parts"], nan(most, heads, D) if chunk else None)
            decay = None
        ops.gla_scan(proj, *self.off[:3], decay, self.q_scale, heads, D, E, state, q_start, slots, n, parts, chunk,
                     nan(most, heads, D, E) if chunk else None, nan(most, heads, D) if chunk else None, **kind)
        ops.gla_output(parts, heads, D, E, weight, self.eps, proj, self.off[3], out, self.gate, 0, **norm)
        return out


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("how", ["scan", 16, 32, "chunks"])
@pytest.mark.parametrize("kind", ["decay", "bonus", "memory"])
@pytest.mark.parametrize("heads,D,E", [(2, 16, 16), (3, 24, 40), (1, 9, 8), (2, 64, 64), (1, 128, 128), (2, 48, 72), (1, 80, 256),
                                       (4, 32, 24), (1, 7, 136)])
def test_recurrences_in_portions_with_states_in_slots(backend, kind, how, heads, D, E):
    """Three requests of unequal length in one call, then their next portions (one of two rows) in a
    second one from the states the first left in scattered slots, against the plain recurrence over
    the whole sequences: row by row, in chunks that run side by side, and as products of 64-row chunks
    (chunks that end inside a request's rows, requests shorter than a chunk)."""
    ops = ops_of(backend)
    dev = ops.device
    r = Recurrence(kind, heads, D, E, [197, 5, 64], seed=3)
    state = torch.zeros(6, heads, D, E, device=dev)
    state[4] = 9.0                                   # (a slot nobody uses stays as it is)
    norm_state = torch.zeros(6, heads, D, device=dev)
    slots = ints([3, 0, 5], dev)
    cut = [90, 3, 2]
    for part in (0, 1):
        spans = [(0, c) if part == 0 else (c, n) for c, n in zip(cut, r.lengths)]
        out = r.step(ops, spans, slots, state, norm_state, how, torch.float32)
        want = torch.cat([r.want[b][lo:hi] for b, (lo, hi) in enumerate(spans)])
        close(out, want, torch.float32, f"part {part}", f32=1e-4)
    for b, slot in enumerate((3, 0, 5)):
        last = r.last[b][0] if kind == "memory" else r.last[b]
        close(state[slot], last, torch.float32, f"state of request {b}", f32=3e-5)
        if kind == "memory":
            close(norm_state[slot], r.last[b][1], torch.float32, f"normaliser of request {b}", f32=3e-5)
    assert float((state[4] - 9.0).abs().max()) == 0.0


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("kind", ["decay", "bonus", "memory"])
@pytest.mark.parametrize("how", ["scan", "chunks"])
def test_recurrences_with_harsh_decays(backend, kind, how):
    """Decays from nothing kept (logarithms of -10,000 and below) to nothing forgotten, row by row and
    channel by channel: no overflow, nothing leaks past a row that forgets everything."""
    ops = ops_of(backend)
    dev = ops.device
    r = Recurrence(kind, 2, 40, 48, [150, 40], seed=5, harsh=True)
    state, norm_state = torch.zeros(2, 2, 40, 48, device=dev), torch.zeros(2, 2, 40, device=dev)
    out = r.step(ops, [(0, 150), (0, 40)], ints([0, 1], dev), state, norm_state, how, torch.float32)
    close(out, torch.cat(r.want), torch.float32, "outputs", f32=1e-4)


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind", ["decay", "bonus", "memory"])
@pytest.mark.parametrize("heads,D,E,rank", [(2, 16, 16, 16), (3, 24, 40, 3), (1, 9, 8, 5), (2, 64, 128, 64), (1, 128, 128, 16),
                                            (4, 32, 24, 7), (1, 60, 512, 8)])
def test_one_row_of_a_recurrence_whole(backend, dtype, kind, heads, D, E, rank):
    """Single rows one after the other through the launch that decoding takes, from the projections to
    the gated output, two requests side by side, against the plain mixers' equations."""
    ops = ops_of(backend)
    dev = ops.device
    assert ops.__class__.__name__ == "EmuOps" or ops.recurrent_row_takes(D, E, rank)
    hd, he, n = heads * D, heads * E, 5
    off = (2, 2 + hd, 2 + 2 * hd, 2 + 2 * hd + he)
    off_low = 2 + 2 * hd + 2 * he
    proj = [randn(n, off_low + max(rank, 2 * heads) + 3, seed=1 + b) for b in range(2)]
    weight = 1.0 + randn(E if kind == "decay" else he, seed=4, scale=0.3)
    w2, bias, bonus = randn(hd, rank, seed=5, scale=0.5), randn(hd, seed=6), randn(hd, seed=7)
    bi, bf = randn(heads, seed=8), 1.0 + randn(heads, seed=9)
    state, norm_state, max_state = (torch.zeros(*s, device=dev) for s in ((4, heads, D, E), (4, heads, D), (4, heads)))
    wants = []
    for b in range(2):
        p = proj[b].to(F64)
        q, k = (p[:, o:o + hd].view(n, heads, D) for o in off[:2])
        q, v = 0.4 * q, p[:, off[2]:off[2] + he].view(n, heads, E)
        low = p[:, off_low:off_low + rank]
        if kind == "memory":
            i = 5.0 * torch.tanh((p[:, off_low:off_low + heads] + bi) / 5.0)
            f = torch.nn.functional.logsigmoid(5.0 * torch.tanh((p[:, off_low + heads:off_low + 2 * heads] + bf) / 5.0))
            o = P.matrix_memory(q, k, v, i, f)[0]
        elif kind == "bonus":
            w = torch.exp(-torch.exp(torch.tanh(low) @ w2.to(F64).T + bias)).view(n, heads, D)
            o = P.bonus_rule(q, k, v, w, bonus.to(F64).view(heads, D))[0]
        else:
            o = P.decay_rule(q, k, v, (torch.sigmoid(low @ w2.to(F64).T + bias) ** 0.2).view(n, heads, D))[0]
        g = p[:, off[3]:off[3] + he]
        w = weight.to(F64).repeat(heads) if kind == "decay" else weight.to(F64)
        wants.append(P.unit_rms(o, 1e-5).reshape(n, he) * w * (torch.sigmoid(g) if kind == "memory" else P.silu(g)))
    to = lambda x: x.to(dev)
    if kind == "memory":
        how = dict(memory=(off_low, off_low + heads, to(bi), to(bf), 5.0, norm_state, max_state))
    else:
        how = dict(decay=(off_low, rank, to(w2), to(bias), "double_exp" if kind == "bonus" else "sigmoid", 5.0))
        if kind == "bonus":
            how["bonus"] = to(bonus)
    for t in range(n):
        rows = torch.cat([proj[0][t:t + 1], proj[1][t:t + 1]]).to(dev)
        out = torch.full((2, he), float("nan"), dtype=dtype, device=dev)
        ops.recurrent_row(rows, *off, 0.4, heads, D, E, state, ints([0, 1, 2], dev), ints([2, 1], dev), 2, to(weight), 1e-5,
                          "sigmoid" if kind == "memory" else "silu", 0, out, **how)
        close(out, torch.cat([wants[0][t:t + 1], wants[1][t:t + 1]]), dtype, f"row {t}", f32=5e-5)
    assert float(state[[0, 3]].abs().max()) == 0.0


def test_the_memory_s_running_maximum_starts_at_zero():
    """The oracle's own sense: a first row with a tiny input gate is divided by the floor exp(-m) of a maximum
    that starts at 0, so its output is small; from minus infinity it would come out at full size."""
    q = k = torch.ones(1, 1, 4, dtype=F64)
    v = torch.full((1, 1, 3), 2.0, dtype=F64)
    out, (_, n, m) = P.matrix_memory(q, k, v, torch.full((1, 1), -5.0, dtype=F64), torch.zeros(1, 1, dtype=F64))
    assert float(m) == 0.0
    assert abs(float(out[0, 0, 0]) - 2.0 * 4.0 * math.exp(-5.0) / (1.0 + 1e-6)) < 1e-9


def test_sizes_that_are_not_taken_go_to_the_scan():
    """States too wide for a chunk's products or for one row's registers fall back, by the rules."""
    emu = ops_of("emu")
    assert not emu.chunk_scan_takes(8, 64, 64)


@pytest.mark.gpu
def test_what_the_kernels_take():
    ops = ops_of("hip")
    assert ops.chunk_scan_takes(32, 128, 256) and not ops.chunk_scan_takes(31, 64, 64)
    assert not ops.chunk_scan_takes(64, 129, 64) and not ops.chunk_scan_takes(64, 64, 264)
    assert ops.recurrent_row_takes(64, 512) and not ops.recurrent_row_takes(256, 512) and not ops.recurrent_row_takes(64, 66)
    assert not ops.recurrent_row_takes(64, 64, 600)
