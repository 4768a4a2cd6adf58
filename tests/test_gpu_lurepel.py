"""Lurepel on the GPU: every new kernel, and every new turn of an older one, alone against the plain implementation's function
of the same mechanism; the engine over every cut of the work (whole prompts, token by token, portions down to two tokens, batches
of unequal requests, slots and pages used again) in float32 and bfloat16 on configurations that differ in every size; models in
which ONE key decides the logits, far back, at page borders, at the first positions and just inside and just outside a chunk, in
a prompt and decoded; long decoding through the captured steps; greedy generation through the entry point and the trace replay
program."""

import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import lurepel_models as lm
import plain_lurepel as plain
import schedules
from test_gpu_pudorax import STRAY, TOLERANCE, check, check_each, dev, engine_for, rel, rounded, tol, tolerances_for

pytestmark = pytest.mark.gpu

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
DTYPES = [torch.float32, torch.bfloat16]
PAGE = 64


@pytest.fixture(scope="module")
def K():
    from beholdd.kernels import HipKernels
    return HipKernels("cuda:0")


# ---- kernels alone ------------------------------------------------------------------------------------------

@pytest.mark.parametrize("w_dtype", DTYPES)
@pytest.mark.parametrize("rows,width,blocks", [(1, 48, 0), (33, 1000, 0), (8, 4096, 8), (3, 8192, 16), (70, 2048, 16), (300, 4096, 0), (5, 9001, 0)])
def test_add_rmsnorm(K, w_dtype, rows, width, blocks):
    """The residual plus the normed result, in place, and the rounded copy in rows or in a product's blocks."""
    from beholdd.kernels.library import BlockedRows
    rng = np.random.default_rng(width)
    h, y = rng.standard_normal((rows, width)).astype(np.float32) * 4, rng.standard_normal((rows, width)).astype(np.float32) * 0.01
    w_t, w = rounded(1 + 0.3 * rng.standard_normal(width), w_dtype)
    want = h + plain.norm(y, w, 1e-5)
    for out in (None, torch.empty(rows, width, device="cuda:0"), torch.empty(rows, width, dtype=torch.bfloat16, device="cuda:0"),
                K._new_blocked(rows, width, blocks) if blocks else None):
        hidden = dev(h)
        K.add_rmsnorm(hidden, dev(y), dev(w_t), 1e-5, out)
        assert rel(hidden, want) < 2e-6
        if out is None:
            continue
        if isinstance(out, BlockedRows):
            out = K.from_blocked(out)
        assert torch.equal(out, hidden.to(out.dtype))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("packed", [False, True])
@pytest.mark.parametrize("m,width,k", [(1, 96, 64), (8, 256, 512), (20, 128, 1024), (40, 8192, 1024), (64, 1024, 512), (90, 4096, 512), (130, 512, 256),
                                       (300, 1024, 256), (700, 4096, 256), (7, 50, 72), (33, 40, 40)])
def test_gelu_gate_in_every_gated_product(K, dtype, packed, m, width, k):
    """gelu(a Wg^T) * (a Wu^T) in the epilogue of every product that carries a gate: few rows, the shared-activation kernel with
    and without parts, tiles, K in parts, the kernel of many rows; sizes that take no fused product."""
    rng = np.random.default_rng(m + width)
    a_t, a = rounded(rng.standard_normal((m, k)), dtype)
    w_t, w = rounded(rng.standard_normal((2 * width, k)) * 2 / np.sqrt(k), dtype)
    weight = K.pack_weight(dev(w_t)) if packed else dev(w_t)
    out = torch.empty(m, width, dtype=dtype, device="cuda:0")
    K.gemm_swiglu(dev(a_t), weight, out, gate="gelu_tanh")
    both = plain.linear(a, w)
    want = plain.gelu(both[:, :width]) * both[:, width:]
    # (the form without a fused product rounds both halves to bfloat16 ahead of the gate)
    assert rel(out, want) < tol(dtype, f32=2e-5, bf16=1.2e-2)
    K.gemm_swiglu(dev(a_t), weight, out)
    assert rel(out, plain.silu(both[:, :width]) * both[:, width:]) < tol(dtype, f32=2e-5, bf16=1.2e-2)
    reader = K.new_rows(m, width, dtype, 2 * width)
    K.gemm_swiglu(dev(a_t), weight, reader, gate="gelu_tanh")
    got = K.from_blocked(reader) if not isinstance(reader, torch.Tensor) else reader
    assert rel(got, want) < tol(dtype, f32=2e-5, bf16=1.2e-2)


def test_gelu_gate_far_from_zero(K):
    z = np.concatenate([np.linspace(-40, 40, 401), [-1e4, 1e4, 0.0, -0.0, 1e-20]]).astype(np.float32)
    both = dev(np.concatenate([z[None], np.ones_like(z)[None]], axis=1))
    out = torch.empty(1, len(z), device="cuda:0")
    K.swiglu(both, out, "gelu_tanh")
    got, want = out.cpu().numpy()[0], plain.gelu(z)
    assert np.isfinite(got).all() and np.abs(got - want).max() < 2e-6 * np.abs(want).max() and np.abs((got - want)[np.abs(z) < 6]).max() < 2e-6


class Layout:
    def __init__(self, lengths, pasts):
        self.n_seqs, self.max_rows_per_seq = len(lengths), max(lengths)
        self.max_position = max(p + n for p, n in zip(pasts, lengths)) - 1
        self.seq_start = dev(np.concatenate([[0], np.cumsum(lengths)]).astype(np.int32))


def paged(lengths, kv_heads, pad, dtype, rng):
    """Pages for sequences of these lengths (scattered over more pages than are needed, which hold other numbers), their table."""
    counts = [-(-n // PAGE) for n in lengths]
    total = sum(counts) + 2
    k_pages = torch.full((total, kv_heads, PAGE, pad), 3.0, dtype=dtype, device="cuda:0")
    v_pages = torch.full((total, kv_heads, pad, PAGE), -2.0, dtype=dtype, device="cuda:0")
    order, at = rng.permutation(total).astype(np.int32), 0
    table = np.zeros((len(lengths), max(counts) + 1), np.int32)
    for row, count in enumerate(counts):
        table[row, :count] = order[at:at + count]
        at += count
    return k_pages, v_pages, dev(table)


ATTENTION = [  # heads, kv_heads, dim, pad, turned, base, slowed, chunk, window, lengths
    (4, 2, 32, 32, 16, 500.0, (4.0, 1.0, 4.0, 64), 70, 0, [150, 3, 64]),
    (8, 1, 96, 96, 96, 1000.0, None, 64, 0, [130, 65]),
    (3, 3, 20, 32, 6, 50.0, (8.0, 1.0, 2.0, 32), 0, 0, [77, 1]),
    (2, 1, 160, 160, 32, 3e4, (2.0, 1.0, 8.0, 128), 200, 0, [420]),
    (16, 1, 64, 64, 0, 1.0, None, 1, 0, [70, 5]),
    (17, 1, 128, 128, 128, 1e6, (8.0, 1.0, 4.0, 256), 128, 0, [129, 256, 300]),
    (16, 4, 128, 128, 64, 1e5, (8.0, 1.0, 4.0, 256), 8192, 0, [1200]),
    (4, 2, 64, 64, 64, 1e4, None, 0, 65, [200, 66]),
]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,kv_heads,dim,pad,turned,base,slowed,chunk,window,lengths", ATTENTION)
def test_attention_over_keys_that_are_values(K, dtype, heads, kv_heads, dim, pad, turned, base, slowed, chunk, window, lengths):
    """From projected rows to gated heads, for whole sequences: unit heads, turned neighbours, raw keys as values, a term of score 0
    in every sum, chunks or a window, a gate a head.  Then the sequences' last rows once more as a decode step, in the two
    launches and in the one that does it all, over pages that lack them; and every one of them writes the same pages."""
    from beholdd.parts.rope import RotaryFrequencies
    rng = np.random.default_rng(dim + heads)
    eps, scale, first = 1e-5, 3.0 / np.sqrt(dim), 8
    total = sum(lengths)
    width = first + (heads + kv_heads) * dim + heads
    width += -width % 8
    rows_t, rows = rounded(rng.standard_normal((total, width)), dtype)
    gate_first = first + (heads + kv_heads) * dim
    rotation = RotaryFrequencies(turned, base, slowed=slowed) if turned else None
    rot = lm.rotation(turned, base, slowed) if turned else None
    starts = np.concatenate([[0], np.cumsum(lengths)])
    want, keys_want = np.zeros((total, heads, dim)), np.zeros((total, kv_heads, dim))
    for s, n in enumerate(lengths):
        mine = rows[starts[s]:starts[s + 1]]
        q = mine[:, first:first + heads * dim].reshape(n, heads, dim)
        k = mine[:, first + heads * dim:gate_first].reshape(n, kv_heads, dim)
        v = k
        if rot:
            q, k = plain.turn(q, np.arange(n), rot), plain.turn(k, np.arange(n), rot)
        q, k = plain.unit(q, eps), plain.unit(k, eps)
        seen = plain.seen(n, chunk)
        if window:
            seen &= np.arange(n)[:, None] - np.arange(n)[None, :] < window
        gates = plain.sigmoid(mine[:, gate_first:gate_first + heads])
        want[starts[s]:starts[s + 1]] = plain.attend(q, k, v, scale, seen) * gates[:, :, None]
    sinks = torch.zeros(heads, device="cuda:0")
    freq = rotation.frequencies("cuda:0") if rotation else None

    def write(rows_dev, positions, row_seq, q_out, pages):
        K.head_norm_rope_write(rows_dev, first, None, None, None, eps, freq, turned, positions, row_seq, q_out, *pages, heads, kv_heads, dim, dim, pad,
                               True, neighbours=True, unit_norm=True, values_are_keys=True)

    positions = dev(np.concatenate([np.arange(n) for n in lengths]).astype(np.int32))
    row_seq = dev(np.repeat(np.arange(len(lengths)), lengths).astype(np.int32))
    pages = paged(lengths, kv_heads, pad, dtype, rng)
    q_out = torch.empty(total, heads * pad, dtype=dtype, device="cuda:0")
    write(dev(rows_t), positions, row_seq, q_out, pages)
    attended = torch.empty(total, heads * pad, dtype=dtype, device="cuda:0")
    span = dict(window=window, chunk=chunk)
    K.attention(q_out, attended, *pages, row_seq, positions, heads, kv_heads, pad, scale, layout=Layout(lengths, [0] * len(lengths)), sinks=sinks,
                gates=dev(rows_t), gate_first=gate_first, **span)
    got = attended.float().reshape(total, heads, pad)
    assert rel(got[..., :dim], want) < tol(dtype, f32=3e-5, bf16=1.6e-2)
    assert pad == dim or float(got[..., dim:].abs().max()) == 0.0
    # the last rows as a decode step
    last = starts[1:] - 1
    last_rows, last_positions = dev(rows_t[torch.from_numpy(last)]), dev((np.asarray(lengths) - 1).astype(np.int32))
    decode_seq = dev(np.arange(len(lengths), dtype=np.int32))
    layout = Layout([1] * len(lengths), [n - 1 for n in lengths])
    before = rows_t.clone()
    before[torch.from_numpy(last)] = 9.0                      # what the pages hold there must not matter
    results = []
    for one_launch in (False, True):
        rng2 = np.random.default_rng(dim + heads + 1)
        pages = paged(lengths, kv_heads, pad, dtype, rng2)
        write(dev(before), positions, row_seq, torch.empty_like(q_out), pages)
        out = torch.empty(len(lengths), heads * pad, dtype=dtype, device="cuda:0")
        common = dict(sinks=sinks, gates=last_rows, gate_first=gate_first, **span)
        if one_launch:
            cos = sin = None
            if rotation:
                cos, sin = (torch.empty(len(lengths), turned // 2, device="cuda:0") for _ in range(2))
                K.row_angles(last_positions, freq, 1.0, cos, sin)
                angle = (np.asarray(lengths, np.float64) - 1)[:, None] * plain.frequencies(rot)[None]
                assert rel(cos, np.cos(angle)) < 2e-4 and rel(sin, np.sin(angle)) < 2e-4
            took = pad == dim and K.attention_decode_pairs(last_rows, first, out, None, None, eps, cos, sin, last_positions, *pages, heads, kv_heads, pad,
                                                           scale, True, layout, unit_norm=True, values_are_keys=True, **common)
            assert took == (dtype == torch.bfloat16 and pad == dim and heads // kv_heads <= 16)
            if not took:
                continue
        else:
            q_last = torch.empty(len(lengths), heads * pad, dtype=dtype, device="cuda:0")
            write(last_rows, last_positions, decode_seq, q_last, pages)
            K.attention(q_last, out, *pages, decode_seq, last_positions, heads, kv_heads, pad, scale, layout=layout, **common)
        assert rel(out.float().reshape(len(lengths), heads, pad)[..., :dim], want[last]) < tol(dtype, f32=3e-5, bf16=1.6e-2), one_launch
        results.append(pages)
    if len(results) == 2:
        assert torch.equal(results[0][1], results[1][1])                                       # the values: copies
        assert rel(results[0][0].float(), results[1][0].double().cpu().numpy()) < 8e-3          # the keys: normed before or after the turn


def test_one_launch_decode_with_norm_weights_and_values_of_their_own(K):
    """The same launch for heads whose norm has weights and whose rows hold values: held to the two launches."""
    from beholdd.parts.rope import RotaryFrequencies
    rng = np.random.default_rng(8)
    heads, kv_heads, dim, n, past, dtype = 8, 2, 64, 5, 130, torch.bfloat16
    rotation = RotaryFrequencies(32, 1000.0, (4.0, 64, 16.0, 1.0))
    freq = rotation.frequencies("cuda:0")
    wq, wk = (dev((1 + 0.3 * rng.standard_normal(dim)).astype(np.float32)) for _ in range(2))
    old = dev(torch.from_numpy(rng.standard_normal((n * past, (heads + 2 * kv_heads) * dim)).astype(np.float32)).to(dtype))
    new = dev(torch.from_numpy(rng.standard_normal((n, (heads + 2 * kv_heads) * dim)).astype(np.float32)).to(dtype))
    positions, row_seq = dev(np.tile(np.arange(past), n).astype(np.int32)), dev(np.repeat(np.arange(n), past).astype(np.int32))
    at, seq = dev(np.full(n, past, np.int32)), dev(np.arange(n, dtype=np.int32))
    outs = []
    for one_launch in (False, True):
        pages = paged([past + 1] * n, kv_heads, dim, dtype, np.random.default_rng(1))
        scrap = torch.empty(n * past, heads * dim, dtype=dtype, device="cuda:0")
        form = dict(neighbours=True, magnitude=rotation.magnitude)
        K.head_norm_rope_write(old, 0, None, wq, wk, 1e-5, freq, 32, positions, row_seq, scrap, *pages, heads, kv_heads, dim, dim, dim, True, **form)
        out = torch.empty(n, heads * dim, dtype=dtype, device="cuda:0")
        if one_launch:
            cos, sin = (torch.empty(n, 16, device="cuda:0") for _ in range(2))
            K.row_angles(at, freq, rotation.magnitude, cos, sin)
            assert K.attention_decode_pairs(new, 0, out, wq, wk, 1e-5, cos, sin, at, *pages, heads, kv_heads, dim, 0.125, True, Layout([1] * n, [past] * n), window=100)
        else:
            q = torch.empty(n, heads * dim, dtype=dtype, device="cuda:0")
            K.head_norm_rope_write(new, 0, None, wq, wk, 1e-5, freq, 32, at, seq, q, *pages, heads, kv_heads, dim, dim, dim, True, **form)
            K.attention(q, out, *pages, seq, at, heads, kv_heads, dim, 0.125, 100, layout=Layout([1] * n, [past] * n))
        outs.append((out, *pages[:2]))
    assert rel(outs[1][0], outs[0][0].double().cpu().numpy()) < 1.6e-2
    assert torch.equal(outs[0][2], outs[1][2]) and torch.equal(outs[0][1], outs[1][1])


@pytest.mark.parametrize("n_seqs,context,chunk,window", [(1, 5000, 1024, 0), (8, 3000, 700, 0), (2, 9000, 0, 0), (3, 4100, 4096, 0), (1, 6000, 0, 1500)])
def test_few_sequences_with_long_contexts_in_key_splits(K, n_seqs, context, chunk, window):
    """Decode rows whose keys go over several workgroups, chunks and windows shorter than the context among them: the walk over a
    stretch of keys is cut by the stretch's pages, and sink and gates are applied once, where the parts are joined."""
    rng = np.random.default_rng(context)
    heads, kv_heads, dim, dtype, scale = 8, 2, 64, torch.bfloat16, 0.25
    lengths = [context - 37 * s for s in range(n_seqs)]
    k_t, k = rounded(rng.standard_normal((n_seqs, context, kv_heads, dim)), dtype)
    rows_t, rows = rounded(rng.standard_normal((n_seqs, heads * dim + kv_heads * dim + heads)), dtype)
    pages = paged(lengths, kv_heads, dim, dtype, rng)
    for s, n in enumerate(lengths):
        packed = torch.cat([torch.zeros(n, heads * dim, dtype=dtype), k_t[s, :n].reshape(n, -1)], dim=1)
        packed[n - 1, heads * dim:] = rows_t[s, heads * dim:heads * dim + kv_heads * dim]
        K.head_norm_rope_write(dev(packed), 0, None, None, None, 1e-5, None, 0, dev(np.arange(n, dtype=np.int32)), dev(np.full(n, s, np.int32)),
                               torch.empty(n, heads * dim, dtype=dtype, device="cuda:0"), *pages, heads, kv_heads, dim, dim, dim, True,
                               unit_norm=True, values_are_keys=True)
    want = np.zeros((n_seqs, heads, dim))
    for s, n in enumerate(lengths):
        values = k[s, :n].copy()
        values[n - 1] = rows[s, heads * dim:heads * dim + kv_heads * dim].reshape(kv_heads, dim)
        q = plain.unit(rows[s:s + 1, :heads * dim].reshape(1, heads, dim), 1e-5)
        lo = (n - 1) - (n - 1) % chunk if chunk else max(0, n - window) if window else 0
        visible = (np.arange(n) >= lo)[None]
        want[s] = plain.attend(q, plain.unit(values, 1e-5), values, scale, visible)[0] * plain.sigmoid(rows[s, -heads:])[:, None]
    positions = dev((np.asarray(lengths) - 1).astype(np.int32))
    out = torch.empty(n_seqs, heads * dim, dtype=dtype, device="cuda:0")
    layout = Layout([1] * n_seqs, [n - 1 for n in lengths])
    common = dict(sinks=torch.zeros(heads, device="cuda:0"), gates=dev(rows_t), gate_first=heads * dim + kv_heads * dim, window=window, chunk=chunk)
    assert K.attention_decode_pairs(dev(rows_t), 0, out, None, None, 1e-5, None, None, positions, *pages, heads, kv_heads, dim, scale, True, layout,
                                    unit_norm=True, values_are_keys=True, **common)
    assert rel(out.float().reshape(n_seqs, heads, dim), want) < 1.6e-2
    q = torch.empty(n_seqs, heads * dim, dtype=dtype, device="cuda:0")
    q.copy_(torch.from_numpy(plain.unit(rows[:, :heads * dim].reshape(n_seqs, heads, dim), 1e-5).reshape(n_seqs, -1).astype(np.float32)))
    K.attention(q, out, *pages, dev(np.arange(n_seqs, dtype=np.int32)), positions, heads, kv_heads, dim, scale, layout=layout, **common)
    assert rel(out.float().reshape(n_seqs, heads, dim), want) < 1.6e-2


@pytest.mark.parametrize("rows,experts,top", [(1, 1, 1), (37, 10, 2), (5, 64, 32), (70, 300, 8), (9, 1000, 4)])
def test_routing_by_corrected_softmax_scores(K, rows, experts, top):
    rng = np.random.default_rng(experts)
    z, correction = (rng.standard_normal((rows, experts)) * 2).astype(np.float32), (rng.standard_normal(experts) * 0.2).astype(np.float32)
    for use in (correction, None):
        chosen, weights = torch.empty(rows, top, dtype=torch.int32, device="cuda:0"), torch.empty(rows, top, device="cuda:0")
        K.route_top_k(dev(z), None, chosen, weights, scoring="softmax_all", correction=None if use is None else dev(use))
        w = {"m.router": np.eye(experts), "m.correction": np.zeros(experts) if use is None else use}
        want, shares = plain.route(z, w, "m.", top)
        choice = np.sort(plain.softmax(z.astype(np.float64)) + w["m.correction"], axis=-1)
        sure = np.ones(rows, bool) if top == experts else (np.diff(choice[:, -top - 1:], axis=-1).min(axis=-1) > 1e-6)
        assert sure.mean() > 0.7
        assert np.array_equal(chosen.cpu().numpy()[sure], want[sure]) and rel(weights[torch.from_numpy(sure)], shares[sure]) < 1e-5
    tied = torch.zeros(3, experts, device="cuda:0")                       # equal scores: the lower index
    chosen, weights = torch.empty(3, top, dtype=torch.int32, device="cuda:0"), torch.empty(3, top, device="cuda:0")
    K.route_top_k(tied, None, chosen, weights, scoring="softmax_all")
    assert chosen.cpu().numpy().tolist() == [list(range(top))] * 3 and rel(weights, np.full((3, top), 1.0 / experts)) < 1e-6


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows,width,experts,identity,top,ff", [(1, 64, 4, 2, 1, 40), (37, 192, 8, 3, 3, 96), (5, 130, 5, 1, 6, 33), (700, 256, 16, 4, 2, 64),
                                                                (300, 128, 4, 4, 1, 128), (260, 72, 2, 6, 2, 24), (64, 1024, 8, 8, 4, 256)])
def test_experts_some_of_which_hand_their_input_through(K, dtype, rows, width, experts, identity, top, ff):
    """The part with its forms (pair by pair for odd sizes, an expert's rows at once, products over gathered rows, in one launch and
    one by one) against the plain experts, written over what stood there and added to it; scratch memory that holds nothing
    finite must not reach a row."""
    from beholdd.parts.base import StepContext
    from beholdd.parts.experts import RoutedExperts
    rng = np.random.default_rng(rows + experts)
    h_t, h = rounded(rng.standard_normal((rows, width)), dtype)
    names = {"m.router": rng.standard_normal((experts + identity, width)) * 3 / np.sqrt(width), "m.correction": rng.standard_normal(experts + identity) * 0.1}
    for e in range(experts):
        names.update({f"m.e{e}.gate": rng.standard_normal((ff, width)) / np.sqrt(width) * 2, f"m.e{e}.up": rng.standard_normal((ff, width)) / np.sqrt(width) * 2,
                      f"m.e{e}.down": rng.standard_normal((width, ff)) / np.sqrt(ff)})
    names = {k: rounded(v, dtype)[1] for k, v in names.items()}
    part = RoutedExperts(width, experts, top, ff, float("inf"), "m.", alpha=1.0, router_bias=False, scoring="softmax_all", shift=0.0, identity=identity,
                         correction=True)
    part.load(lambda name: dev(names[name], dtype))
    part.prepare(K)
    mlp = {"router": {"experts": experts, "identity": identity, "top": top}}
    want = plain.experts(h, names, "m.", mlp)
    chosen, shares = plain.route(h, names, "m.", top)
    assert (chosen >= experts).any() or rows == 1
    choice = np.sort(plain.softmax(plain.linear(h, names["m.router"])) + names["m.correction"], axis=-1)
    sure = torch.from_numpy(choice[:, -top] - choice[:, -top - 1] > 1e-4 if top < experts + identity else np.ones(rows, bool))
    for is_decode, one_launch in ((True, None), (False, True), (False, False)):
        if one_launch is False:
            part.in_one_launch = False
        part.ONE_LAUNCH_WORK = 1e30
        ctx = StepContext(kernels=K, act_dtype=dtype, device=torch.device("cuda:0"), n_rows=rows, n_seqs=rows if is_decode else 1, tokens=None,
                          positions=None, row_seq=None, seq_start=None, seq_slot=None, seq_past=None, host_seq_start=[], host_seq_slot=[],
                          host_seq_past=[], is_decode=is_decode, max_position=0)
        poison = [torch.full((rows * top * max(width, 2 * ff),), float("nan"), device="cuda:0") for _ in range(3)]
        del poison                                       # the allocator hands this memory out again
        for fresh in (True, False):
            hidden = torch.full((rows, width), 5.0, device="cuda:0")
            part.forward(ctx, dev(h_t), hidden, fresh=fresh)
            assert rel(hidden[sure], (want + (0.0 if fresh else 5.0))[sure.numpy()]) < tol(dtype, f32=5e-5, bf16=2e-2), (is_decode, one_launch, fresh)
        got_chosen, got_shares = ctx.extras["routing"]
        assert rel(got_shares.sort(dim=-1).values[sure], np.sort(shares[sure.numpy()], axis=-1)) < 1e-5


@pytest.mark.parametrize("rows,experts,top,width,ff", [(1, 3, 1, 64, 16), (8, 32, 4, 2048, 768), (40, 2, 2, 256, 80), (33, 5, 3, 4096, 48), (5, 1, 1, 192, 1536)])
@pytest.mark.parametrize("weighed", [False, True])
def test_experts_of_few_rows_on_the_matrix_cores(K, rows, experts, top, width, ff, weighed):
    """Both products of `experts_tiles` against the plain ones: experts without pairs, with more than sixteen (several passes over the
    matrix), chunks that do not divide evenly over the waves; the gate's clamp and offset and a weight on the input."""
    rng = np.random.default_rng(rows * experts)
    x_t, x = rounded(rng.standard_normal((rows, width)), torch.bfloat16)
    gu_t, gu = rounded(rng.standard_normal((experts, 2 * ff, width)) * 2 / np.sqrt(width), torch.bfloat16)
    down_t, down = rounded(rng.standard_normal((experts, width, ff)) / np.sqrt(ff), torch.bfloat16)
    chosen = np.stack([rng.permutation(experts)[:top] for _ in range(rows)]).astype(np.int32)
    share = rng.uniform(0.2, 1.0, (rows, top)).astype(np.float32)
    lists, counts = torch.empty(experts, rows, dtype=torch.int32, device="cuda:0"), torch.empty(experts, dtype=torch.int32, device="cuda:0")
    K.experts_group(dev(chosen), lists, counts)
    inner = torch.empty(rows * top, ff, dtype=torch.bfloat16, device="cuda:0")
    K.experts_tiles(dev(x_t), top, lists, counts, K.pack_weight(dev(gu_t.reshape(-1, width))), inner, gated=True, limit=1.5, alpha=1.702, shift=1.0,
                    in_weights=dev(share) if weighed else None)
    want = np.zeros((rows * top, ff))
    for r in range(rows):
        for j in range(top):
            both = gu[chosen[r, j]].astype(np.float64) @ x[r] * (share[r, j] if weighed else 1.0)
            g, u = np.minimum(both[:ff], 1.5), np.clip(both[ff:], -1.5, 1.5)
            want[r * top + j] = g * plain.sigmoid(1.702 * g) * (u + 1.0)
    assert rel(inner, want) < 8e-3
    y = torch.empty(rows * top, width, device="cuda:0")
    if K.experts_tiles_take(torch.bfloat16, ff, width):
        K.experts_tiles(inner, 1, lists, counts, K.pack_weight(dev(down_t.reshape(-1, ff))), y)
    else:
        K.experts_rows(inner, 1, lists, counts, dev(down_t), y)
    held = inner.float().cpu().numpy()
    for p in range(rows * top):
        assert rel(y[p], down[chosen[p // top, p % top]].astype(np.float64) @ held[p]) < 2e-5, p


def test_a_prompt_whose_choices_are_all_identity_experts(K, tmp_path):
    config = {"architecture": "Lurepel", "vocab": 50, "width": 128, "norm": {"eps": 1e-5},
              "layers": [lm.attention(2, 1, 32, 0.3, dims=8, mlp=lm.moe(2, 2, 64, identity=3)), lm.attention(2, 1, 32, 0.3, mlp=lm.dense(64))]}
    weights = lm.random_weights(config, 3)
    weights["l0.mlp.correction"][:] = [-4, -4, 0, 0.5, 0.25]
    folder = lm.write_model(tmp_path / "identity", config, weights)
    requests = schedules.random_requests(50, [90, 3], seed=1)
    want = [plain.forward(config, weights, r) for r in requests]
    for dtype in ("float32", "bfloat16"):
        engine = engine_for(folder, dtype)
        tolerances = tolerances_for(folder, dtype, requests, want)
        check_each("whole", schedules.whole(engine, requests), want, tolerances, STRAY[dtype])
        check_each("tail", schedules.tail_one_by_one(engine, requests, tail=20), want, tolerances, STRAY[dtype])


# ---- the engine over every cut --------------------------------------------------------------------------------------------

@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    made = {}

    def get(name, seed=5):
        if (name, seed) not in made:
            config = lm.CONFIGS[name]
            weights = lm.random_weights(config, seed)
            made[(name, seed)] = (lm.write_model(tmp_path_factory.mktemp(f"lurepel_{name}_{seed}"), config, weights), config, weights)
        return made[(name, seed)]

    return get


LENGTHS = {"mixed": [5, 11, 1, 70, 33, 128, 300], "plain": [1, 7, 23, 64, 90, 200], "odd": [3, 65, 130, 2, 31], "wide": [2, 50, 131, 260]}


@pytest.fixture(scope="module")
def expected(folders):
    cache = {}

    def get(name):
        if name not in cache:
            folder, config, weights = folders(name)
            requests = schedules.random_requests(config["vocab"], LENGTHS[name], seed=11)
            cache[name] = (folder, requests, [plain.forward(config, weights, r) for r in requests])
        return cache[name]

    return get


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", sorted(LENGTHS))
def test_every_cut_matches_the_plain_implementation(expected, name, dtype):
    folder, requests, want = expected(name)
    engine = engine_for(folder, dtype)
    tolerances, stray = tolerances_for(folder, dtype, requests, want), STRAY[dtype]
    whole = schedules.whole(engine, requests)
    check_each("whole", whole, want, tolerances, stray)
    tail = schedules.tail_one_by_one(engine, requests, tail=80)      # past every chunk's edge one token at a time
    check_each("last 80 one by one", tail, want, tolerances, stray)
    for batch_size in (3, len(requests)):
        batched = schedules.batches(engine, requests, batch_size=batch_size)
        check_each(f"batches of {batch_size}", batched, want, tolerances, stray)
    in_portions = schedules.portions(engine, requests)
    check_each("portions", in_portions, want, tolerances, stray)
    pairs = schedules.portions(engine, requests, sizes=(2, 2, 3, 2, 1, 2), rest_every=3)
    check_each("portions of two and three", pairs, want, tolerances, stray)
    between = [t / 2 for t in tolerances] if dtype == "float32" else tolerances
    check_each("tail vs whole", tail, whole, between, stray)
    check_each("batches vs whole", batched, whole, between, stray)
    check_each("portions vs whole", in_portions, whole, between, stray)
    engine.cache.check_invariants()
    assert engine.cache.live_slots() == [] and engine.cache.free_page_count() == engine.cache.n_pages


# Without experts no choice magnifies a rounding: attention and the dense feed-forward are held at every position.
NO_EXPERTS = {
    "architecture": "Lurepel", "vocab": 83, "width": 64, "norm": {"eps": 1e-5},
    "layers": [lm.attention(4, 2, 64, 0.2, chunk=48, dims=16, base=1000.0, slowed=(4.0, 1.0, 4.0, 64), mlp=lm.dense(96)),
               lm.attention(8, 2, 32, 0.25, dims=32, base=300000.0, mlp=lm.dense(40)), lm.attention(2, 2, 96, 0.15, chunk=100)],
}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_every_cut_without_experts_holds_at_every_position(tmp_path, dtype):
    config = NO_EXPERTS
    weights = lm.random_weights(config, 7)
    folder = lm.write_model(tmp_path / "bare", config, weights)
    requests = schedules.random_requests(config["vocab"], [1, 9, 66, 130, 200], seed=21)
    want = [plain.forward(config, weights, r) for r in requests]
    engine = engine_for(folder, dtype)
    tolerances = tolerances_for(folder, dtype, requests, want, least=1e-4 if dtype == "float32" else 3e-2)
    for label, got in (("whole", schedules.whole(engine, requests)), ("tail", schedules.tail_one_by_one(engine, requests, tail=80)),
                       ("batches", schedules.batches(engine, requests, batch_size=3)), ("portions", schedules.portions(engine, requests)),
                       ("small portions", schedules.portions(engine, requests, sizes=(2, 2, 3, 2, 1, 2), rest_every=3))):
        check_each(label, got, want, tolerances, 0.0 if dtype == "float32" else 0.03)
    engine.cache.check_invariants()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_batch_changes_nothing_for_its_members(expected, dtype):
    folder, requests, _ = expected("mixed")
    engine = engine_for(folder, dtype)
    alone = schedules.whole(engine, requests)
    from beholdd.engine import StepEntry
    slots = [engine.alloc_slot() for _ in requests]
    together = engine.step([StepEntry(s, r, list(range(len(r)))) for s, r in zip(slots, requests)]).float().cpu().numpy()
    at = 0
    for r, a in zip(requests, alone):
        check("together", [together[at:at + len(r)]], [a], 2e-5 if dtype == "float32" else TOLERANCE[dtype], STRAY[dtype])
        at += len(r)


# ---- one key decides --------------------------------------------------------------------------------------------------

NEEDLE, ASKER = 7, 9


def one_key_model(tmp_path, chunk, dim, seed=3):
    """One layer whose last query finds ONE key among hundreds: the token NEEDLE alone projects onto a key direction that the
    token ASKER alone asks for (its score stands out by far more than the others' spread; every key has unit length), so the
    asker's logits hang on whether that one position is read."""
    config = {"architecture": "Lurepel", "vocab": 40, "width": 32, "norm": {"eps": 1e-5}, "layers": [lm.attention(2, 1, dim, 20.0 / dim, chunk=chunk, dims=8)]}
    weights = lm.random_weights(config, seed)
    embed = weights["embed"]
    embed[:, :2] = 0.0                        # the other tokens have nothing in the two dimensions that needle and asker use
    embed[NEEDLE] = 0.0
    embed[NEEDLE, 0] = 8.0
    embed[ASKER] = 0.0
    embed[ASKER, 1] = 8.0
    for name in ("embed.norm", "l0.norm1", "final.norm"):
        weights[name][:] = 1.0
    m, at = "l0.mix.", dim - 4                                   # a dimension beyond the turned ones
    weights[m + "q"][:] *= 0.02
    weights[m + "q"][at, 1] = weights[m + "q"][dim + at, 1] = 3.0
    weights[m + "k"][:, 0] = 0.0
    weights[m + "k"][at, 0] = 3.0
    weights[m + "k"][at, 1:] = 0.0                                # nobody else's key has anything there
    weights[m + "g"][:] = 0.0
    weights = {k: lm.bfloat(v) for k, v in weights.items()}
    return lm.write_model(tmp_path / f"one_key_{chunk}_{dim}", config, weights), config, weights


def needle_case(tmp_path, dtype, chunk, needle_at, moves, length=420, dim=32):
    """The needle at `needle_at`, the asker last (at position `length`); `moves`: whether the needle may change the asker's logits."""
    folder, config, weights = one_key_model(tmp_path, chunk, dim)
    rng = np.random.default_rng(needle_at)
    others = [t for t in range(config["vocab"]) if t not in (NEEDLE, ASKER)]
    tokens = [int(rng.choice(others)) for _ in range(length)]
    without = list(tokens) + [ASKER]
    tokens[needle_at] = NEEDLE
    tokens.append(ASKER)
    want, blind = plain.forward(config, weights, tokens)[-1], plain.forward(config, weights, without)[-1]
    if moves:
        assert np.abs(want - blind).max() > 0.2 * np.abs(want).max()             # the one key moves the logits
    else:
        assert np.abs(want - blind).max() < 1e-6 * np.abs(want).max()            # it lies outside what the asker sees
    engine = engine_for(folder, dtype, max_tokens=1024)
    from beholdd.engine import StepEntry
    slot = engine.alloc_slot()
    in_prompt = engine.step([StepEntry(slot, tokens, [len(tokens) - 1])]).float().cpu().numpy()[0]
    engine.free_slot(slot)
    slot = engine.alloc_slot()
    engine.step([StepEntry(slot, tokens[:200], [])])
    engine.step([StepEntry(slot, tokens[200:-3], [])])
    for token in tokens[-3:-1]:
        engine.step([StepEntry(slot, [token], [])])
    decoded = engine.step([StepEntry(slot, tokens[-1:], [0])]).float().cpu().numpy()[0]
    engine.free_slot(slot)
    for got in (in_prompt, decoded):
        assert np.abs(got - want).max() < (1e-4 if dtype == "float32" else 4e-2) * np.abs(want).max()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("needle_at", [0, 1, 63, 64, 65, 127, 128, 300, 419])
def test_one_far_key_decides_where_every_key_is_seen(tmp_path, dtype, needle_at):
    needle_case(tmp_path, dtype, 0, needle_at, True)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("chunk,length", [(64, 420), (96, 430), (130, 420), (2, 421), (65, 419), (141, 422), (420, 500), (210, 419), (7, 384)])
def test_a_key_just_inside_and_just_outside_a_chunk(tmp_path, dtype, chunk, length):
    first = length - length % chunk
    needle_case(tmp_path, dtype, chunk, first, True, length=length, dim=64)            # the first position of the asker's chunk
    needle_case(tmp_path, dtype, chunk, first - 1, False, length=length, dim=64)       # the last of the chunk before
    if length - 1 > first:
        needle_case(tmp_path, dtype, chunk, length - 1, True, length=length, dim=64)   # the neighbour


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("chunk", [64, 70])
def test_a_token_that_opens_a_chunk_sees_itself_alone(tmp_path, dtype, chunk):
    """The asker at a chunk's first position: nothing before it may reach its logits, whatever the pages hold."""
    needle_case(tmp_path, dtype, chunk, 6 * chunk - 1, False, length=6 * chunk)


# ---- long runs, generation, programs ----------------------------------------------------------------------------------

@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_prompts_in_portions_and_long_decoding(folders, dtype):
    """A request of 700 tokens: the prompt in portions that end at, before and after page borders, then 150 tokens one by one
    through the captured steps, in a cache whose pages and slots were used before by other requests."""
    folder, config, weights = folders("wide")
    long_one = schedules.random_requests(config["vocab"], [700], seed=31)[0]
    want = plain.forward(config, weights, long_one)
    engine = engine_for(folder, dtype, max_tokens=1024)
    schedules.whole(engine, schedules.random_requests(config["vocab"], [300, 90], seed=32))
    from beholdd.engine import StepEntry
    slot = engine.alloc_slot()
    rows, at = [], 0
    for size in (63, 1, 64, 65, 127, 2, 100, 128):
        rows.append(engine.step([StepEntry(slot, long_one[at:at + size], list(range(size)))]).float().cpu().numpy())
        at += size
    assert at == 550
    for token in long_one[at:]:
        rows.append(engine.step([StepEntry(slot, [token], [0])]).float().cpu().numpy().copy())
    engine.free_slot(slot)
    tolerance = tolerances_for(folder, dtype, [long_one], [want])[0]
    check("long", [np.concatenate(rows)], [want], tolerance, STRAY[dtype])
    if engine.graphs is not None:
        assert len(engine.graphs.graphs) >= 1          # the one-token steps were captured and replayed
    assert engine.cache.free_page_count() == engine.cache.n_pages


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_greedy_generation_through_the_entry_point(tmp_path, dtype):
    import beholdd
    config = NO_EXPERTS
    weights = lm.random_weights(config, 5, gain=1.5)
    folder = lm.write_model(tmp_path / "generating", config, weights)
    prompts = schedules.random_requests(config["vocab"], [1, 9, 30, 70], seed=6)
    max_new = [12, 9, 12, 40]
    engine = beholdd.Engine(folder, dtype=dtype, max_tokens=1024)
    results = engine.generate(prompts, max_new_tokens=max_new)
    assert len({token for r in results for token in r.token_ids}) >= 6
    for prompt, result, n in zip(prompts, results, max_new):
        assert len(result.token_ids) == n
        if dtype == "float32":
            assert result.token_ids == plain.greedy(config, weights, prompt, n)
            continue
        fed = list(prompt)
        near = 0
        for token in result.token_ids:          # every choice is the plain one's, or lies within rounding of it
            row = plain.forward(config, weights, fed)[-1]
            near += int(row[token] >= row.max() - 0.04 * np.abs(row).max())
            fed.append(token)
        assert near >= 0.9 * n, (near, n)
    sampled = engine.generate(prompts, max_new_tokens=8, temperature=0.9, top_k=20, top_p=0.9, seed=4)
    again = engine.generate(prompts, max_new_tokens=8, temperature=0.9, top_k=20, top_p=0.9, seed=4)
    assert [r.token_ids for r in sampled] == [r.token_ids for r in again]
    engine.cache.check_invariants()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_replay_and_generate_programs(folders, tmp_path, dtype):
    folder, config, weights = folders("odd")
    requests = schedules.random_requests(config["vocab"], [40, 7, 66], seed=9)
    want = [plain.forward(config, weights, r) for r in requests]
    tolerances = tolerances_for(folder, dtype, requests, want)
    steps = schedules.trace_of(schedules.batches, requests, batch_size=3)
    run = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", folder, "--dtype", dtype,
                          "--out", str(tmp_path / "out"), "--max-tokens", "256"],
                         input="\n".join(json.dumps(s) for s in steps) + "\n", capture_output=True, text=True, timeout=600)
    assert run.returncode == 0, run.stderr[-2000:]
    got = [[] for _ in requests]      # every request's rows in the order of its positions, whatever step made them
    for record in steps:
        rows = np.fromfile(tmp_path / "out" / f"{record['step']}.f32", dtype="<f4").reshape(-1, config["vocab"])
        at = 0
        for entry in record["entries"]:
            assert entry["want"] == list(range(len(entry["tokens"])))
            got[int(entry["id"][1:])].append(rows[at:at + len(entry["want"])])
            at += len(entry["want"])
        assert at == len(rows)
    check_each("replayed", [np.concatenate(rows) for rows in got], want, tolerances, STRAY[dtype])
    run = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "beholdd"), "generate", "--model", folder, "--dtype", dtype,
                          "--prompt-ids", ",".join(str(t) for t in requests[1]), "--max-new-tokens", "5"], capture_output=True, text=True, timeout=600)
    assert run.returncode == 0, run.stderr[-2000:]
    if dtype == "float32":
        expected_tokens = plain.greedy(config, weights, requests[1], 5)
        assert all(str(token) in run.stdout for token in expected_tokens), (run.stdout, expected_tokens)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("seed", range(10))
def test_drawn_configurations(seed, dtype, tmp_path):
    """Sizes, counts, constants and layer orders that nobody picked, on the real kernels."""
    config = lm.drawn_config(100 + seed)
    weights = lm.random_weights(config, seed, gain=0.7)
    folder = lm.write_model(tmp_path / "drawn", config, weights)
    requests = schedules.random_requests(config["vocab"], [1, 19, 70, 150], seed=seed)
    want = [plain.forward(config, weights, r) for r in requests]
    engine = engine_for(folder, dtype)
    tolerances, stray = tolerances_for(folder, dtype, requests, want), STRAY[dtype]
    for label, got in (("whole", schedules.whole(engine, requests)), ("tail", schedules.tail_one_by_one(engine, requests, tail=70)),
                       ("batches", schedules.batches(engine, requests, batch_size=3)),
                       ("small portions", schedules.portions(engine, requests, sizes=(2, 2, 3, 2, 1, 2), rest_every=3))):
        check_each(f"{config} {label}", got, want, tolerances, stray)
    engine.cache.check_invariants()
