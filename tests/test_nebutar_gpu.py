"""Nebutar on the GPU: its kernels alone against their stand-ins, and the HIP kernels under the framework's step function,
cache manager, scheduler and entry points, in float32 and bfloat16, against the plain implementation in
``plain_nebutar``: the same small models and cuts as on the CPU, captured decode steps, keys at the edges of chunks, tokens
far back that only the recurrence carries, greedy generation through ``Engine``, the command line and the trace runner as
a user starts it."""

import json
import subprocess
import sys
from pathlib import Path

import numpy as np
import pytest
import torch

import plain_nebutar as plain
from helpers import make_runner, random_prompts, replay, trace_mixed, trace_portions, trace_tail_decode
from nebutar_models import (BLOCK, CUTS, MODELS, check_trace, compare, drawn_model, layer, left, model, moe, oracle, random_weights,
                            read_folder, right, row_errors, with_a_sharp_key, write_model)
from torch_kernels import TorchKernels

pytestmark = pytest.mark.gpu
ROOT = Path(__file__).resolve().parents[1]
DEV = "cuda:0"
DTYPES = {"float32": torch.float32, "bfloat16": torch.bfloat16}
# in units of the logits' spread per position; bfloat16: (every row, nine rows in ten), on weights that settle the choice of
# experts (``settled``): a choice that hangs on less than bfloat16 resolves may fall the other way, and the recurrences
# carry it on to every later token. Choices that depend on the token are compared in float32, and kernel by kernel.
TOL = {"float32": 3e-4, "bfloat16": (0.15, 0.06)}


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    base = tmp_path_factory.mktemp("nebutar_gpu")
    return {(name, dtype): write_model(base / f"{name}_{dtype}", cfg, seed=i + 1, settle=dtype == "bfloat16")
            for i, (name, cfg) in enumerate(MODELS.items()) for dtype in DTYPES}


@pytest.fixture(scope="module")
def kernel_sets():
    from socrates_amd.kernels import HipKernels
    return {name: HipKernels(dt, DEV) for name, dt in DTYPES.items()}


def _close(got, want, dtype, what, scale=1.0):
    tol = dict(atol=2e-5 * scale, rtol=2e-5) if dtype == "float32" else dict(atol=2e-2 * scale, rtol=2e-2)
    torch.testing.assert_close(got.float().cpu(), want.float().cpu(), msg=lambda m: f"{what} ({dtype}): {m}", **tol)


def _ctx(lengths, rows, starts):
    """A step's context for kernels: tokens of several sequences one after the other."""
    from socrates_amd.engine import StepEntry
    from socrates_amd.engine.batch import build_context
    return build_context([StepEntry(r, [0] * n, []) for r, n in zip(rows, lengths)], starts, torch.device(DEV))


# ---- each kernel against its stand-in ----------------------------------------------------------------------
@pytest.mark.parametrize("dtype", list(DTYPES))
@pytest.mark.parametrize("H,G,D,Dv,taps", [(4, 2, 20, 28, 4), (3, 3, 48, 80, 3), (6, 1, 7, 9, 5), (2, 2, 128, 64, 2), (2, 1, 200, 16, 4),
                                           (5, 5, 1, 1, 1), (4, 4, 64, 130, 4), (2, 1, 256, 300, 7), (3, 1, 130, 33, 3), (8, 2, 16, 256, 2)])
@pytest.mark.parametrize("lengths", [[9, 1, 2, 15], [37, 1, 2, 170], [1, 1, 1, 1], [16, 32, 33, 48]])
def test_gated_delta_rule_kernels(kernel_sets, dtype, H, G, D, Dv, taps, lengths):
    """Convolutions, unit vectors, gates and the walk, from inputs and a state that are not zero, several sequences of
    unequal length side by side (single tokens, whole batches of the walk and parts of them), columns of a wider product."""
    ops, dt = kernel_sets[dtype], DTYPES[dtype]
    g = torch.Generator().manual_seed(H * D + Dv)
    ctx = _ctx(lengths, [2, 0, 3, 1], [5, 300, 0, 41])
    N, C, before = ctx.n_tokens, 2 * G * D + H * Dv, 8
    conv_at, at = 4, 4 + ((taps - 1) * C + 3) // 4 * 4
    x = (torch.randn(N, before + C + 5, generator=g) * 0.7).to(dt).to(DEV)
    w = torch.randn(C, taps, generator=g).to(DEV)
    z, a_log, dt_bias = torch.randn(N, 2 * H, generator=g).to(DEV), (torch.randn(H, generator=g) - 1).to(DEV), torch.randn(H, generator=g).to(DEV)
    state = torch.randn(5, (at + H * D * Dv + 7) // 4 * 4, generator=g).to(DEV)
    s1, s2 = state.clone(), state.double().cpu()
    print("delta", dtype, H, G, D, Dv, taps, lengths, flush=True)
    got = ops.delta_rule(x, before, G, H, D, Dv, w, D ** -0.5, 1e-6, z, a_log, dt_bias, s1, conv_at, at, ctx)
    cpu = _ctx_on_cpu(ctx)
    want = TorchKernels(dt, "cpu", acc=torch.float64).delta_rule(x.cpu(), before, G, H, D, Dv, w.cpu(), D ** -0.5, 1e-6, z.cpu(), a_log.cpu(),
                                                                 dt_bias.cpu(), s2, conv_at, at, cpu)
    assert got.dtype == torch.float32
    # (values are rounded to the compute dtype between the two kernels; a state of order one is read through q of length D^-1/2)
    tol = 3e-4 if dtype == "float32" else 2e-2
    torch.testing.assert_close(got.cpu().double(), want, atol=tol * float(want.std()), rtol=tol)
    torch.testing.assert_close(s1.cpu().double(), s2, atol=tol, rtol=tol)
    # rows and places that are not the step's
    assert torch.equal(s1[4], state[4]) and torch.equal(s1[:, :conv_at], state[:, :conv_at]) and torch.equal(s1[:, at + H * D * Dv:], state[:, at + H * D * Dv:])


def _ctx_on_cpu(ctx):
    from types import SimpleNamespace
    return SimpleNamespace(**{k: v.cpu() if isinstance(v, torch.Tensor) else v for k, v in vars(ctx).items()})


@pytest.mark.parametrize("dtype", list(DTYPES))
@pytest.mark.parametrize("d", [1, 5, 40, 96, 1023, 1024, 1536, 2560, 3076, 4096, 4100, 6000, 12000])
@pytest.mark.parametrize("S,N", [(1, 7), (2, 1), (3, 600), (4, 9), (5, 17), (16, 3)])
def test_copies_of_the_stream_kernel(kernel_sets, dtype, d, S, N):
    """New copies from the old ones and one or two branches (rounded, float32, partial sums, experts' results by place with
    choices that hand their input on), and the normed combination with and without a bias, a mean, rows selected."""
    from socrates_amd.kernels.hybrid import ExpertSums
    ops, dt = kernel_sets[dtype], DTYPES[dtype]
    ref = TorchKernels(dt, DEV)
    if N * S * d > 8_000_000:
        pytest.skip("enough at smaller sizes")
    g = torch.Generator().manual_seed(d * 20 + S)
    rnd = lambda *s: torch.randn(*s, generator=g).to(DEV)               # noqa: E731
    x, mix, out, read = rnd(N, S, d), rnd(S, S), rnd(S), rnd(S)
    norms = [(rnd(d), rnd(d), 1e-5, True), (rnd(d), None, 1e-3, False)]
    top, E = 3, 5
    idx = torch.randint(0, E + 2, (N, top), generator=g).to(torch.int32).to(DEV)      # (the last two are identity experts)
    runs = ops.moe_sort(idx, E)
    weight, inp, y = rnd(N, top), rnd(N, d).to(dt), rnd(N * top, d)
    place = runs.place.view(N, top).long()
    assert torch.equal(place < 0, idx >= E)
    by_place = torch.where((place >= 0).unsqueeze(-1), y[place.clamp(min=0)], inp.float().unsqueeze(1))
    summed = (weight.unsqueeze(-1) * by_place).sum(1)
    a, b, parts = rnd(N, d).to(dt), rnd(N, d), rnd(3, N, d)
    cases = [([(a, 1.0)], [(a, 1.0)]), ([(b, 0.3), (parts, -0.7)], [(b, 0.3), (parts, -0.7)]),
             ([(ExpertSums(y, runs, weight, inp), 1.0)], [(summed, 1.0)]), ([(a, 0.5), (b, 2.0)], [(a, 0.5), (b, 2.0)])]
    for k, (mine, theirs) in enumerate(cases):
        norm = norms[k % 2]
        x1, x2 = x.clone(), x.clone()
        print("streams", dtype, d, S, N, k, flush=True)
        got = ops.streams_update(x1, mine, mix, out, read, norm)
        want = ref.streams_update(x2, theirs, mix, out, read, norm)
        # (the copies' sum of some terms: float32 rounding in another order)
        torch.testing.assert_close(x1, x2, atol=2e-4, rtol=2e-5)
        if d > 1:
            _close(got, want, dtype, f"normed combination, case {k}", scale=20.0 if dtype == "float32" else 3.0)
        plain_sum = x.clone()
        assert ops.streams_update(plain_sum, mine, None, None) is None
        torch.testing.assert_close(plain_sum, x + sum(s * (t.sum(0) if t.dim() == 3 else t).float() for t, s in theirs).unsqueeze(1), atol=2e-4, rtol=2e-5)
    rows = torch.randint(0, N, (4,), generator=g).to(torch.int32).to(DEV)
    before = x.clone()
    for norm in norms:
        if d > 1:
            _close(ops.streams_norm(x, read, norm), ref.streams_norm(x, read, norm), dtype, "norm", scale=20.0)
            _close(ops.streams_norm(x, None, norm, rows), ref.streams_norm(x, None, norm, rows), dtype, "norm of rows", scale=20.0)
    assert torch.equal(x, before)
    # the same sum of experts by the kernel that takes it where no block does
    if d % 4 == 0:
        torch.testing.assert_close(ops.moe_combine(y, runs, weight, through=inp), summed, atol=1e-4, rtol=1e-4)


def test_copies_of_the_stream_kernel_refuses_what_does_not_fit(kernel_sets):
    from socrates_amd.kernels import KernelError
    ops = kernel_sets["float32"]
    x, gain = torch.zeros(2, 3, 8, device=DEV), torch.ones(8, device=DEV)
    norm = (gain, None, 1e-5, False)
    for bad in (lambda: ops.streams_norm(torch.zeros(2, 17, 8, device=DEV), None, norm), lambda: ops.streams_norm(x, torch.ones(2, device=DEV), norm),
                lambda: ops.streams_update(x, [], None, None), lambda: ops.streams_update(x, [(torch.zeros(2, 7, device=DEV), 1.0)], None, None),
                lambda: ops.streams_update(x, [(torch.zeros(2, 8, device=DEV), 1.0)], torch.zeros(3, 3, device=DEV), None)):
        with pytest.raises(KernelError):
            bad()


@pytest.mark.parametrize("dtype", list(DTYPES))
def test_embedding_and_choice_of_experts(kernel_sets, dtype):
    ops, dt = kernel_sets[dtype], DTYPES[dtype]
    ref = TorchKernels(dt, DEV)
    g = torch.Generator().manual_seed(8)
    table, pos = torch.randn(37, 21, generator=g).to(dt).to(DEV), torch.randn(50, 21, generator=g).to(dt).to(DEV)
    ids, at = torch.randint(0, 37, (65,), generator=g).to(torch.int32).to(DEV), torch.randint(0, 50, (65,), generator=g).to(torch.int32).to(DEV)
    for n, p in ((1, pos), (3, pos), (2, None)):
        torch.testing.assert_close(ops.embedding_streams(ids, table, -1.5, at, p, n), ref.embedding_streams(ids, table, -1.5, at, p, n))
    for E, top in ((9, 4), (1, 1), (70, 6), (256, 8), (5, 5)):
        z, c = 2 * torch.randn(33, E, generator=g), 0.1 * torch.randn(E, generator=g)
        for scoring in ("softmax", "sigmoid"):
            a = ops.moe_route(z.to(DEV), c.to(DEV), top, scoring=scoring, renorm=False)
            b = ref.moe_route(z.to(DEV), c.to(DEV), top, scoring=scoring, renorm=False)
            assert torch.equal(a[0], b[0])
            torch.testing.assert_close(a[1], b[1], atol=1e-6, rtol=1e-5)
    d, E, same, top, ff = 40, 5, 2, 3, 24
    x = torch.randn(50, d, generator=g).to(dt).to(DEV)
    up, down = (0.3 * torch.randn(E, 2 * ff, d, generator=g)).to(dt).to(DEV), (0.3 * torch.randn(E, d, ff, generator=g)).to(dt).to(DEV)
    idx = torch.stack([torch.randperm(E + same, generator=g)[:top] for _ in range(50)]).to(torch.int32).to(DEV)
    w = torch.rand(50, top, generator=g).to(DEV)
    _close(ops.moe_experts(x, idx, w, up, down, 3e38, 1.0, shift=0.0, identity=True),
           ref.moe_experts(x, idx, w, up, down, 3e38, 1.0, shift=0.0, identity=True), dtype, "experts", scale=10.0)
    # every choice an identity expert: nothing to compute
    only = torch.full((4, 1), E, dtype=torch.int32, device=DEV)
    one = torch.ones(4, 1, device=DEV)
    torch.testing.assert_close(ops.moe_experts(x[:4].contiguous(), only, one, up, down, 3e38, 1.0, shift=0.0, identity=True), x[:4].float())


def _paged(dt, Hkv, P, bs, rows, pages, g, held=None):
    """A slot whose pages hold what no row should see wherever ``held(row, block)`` is false."""
    from socrates_amd.cache.manager import PagedSlot
    table = torch.arange(1, 1 + rows * pages, dtype=torch.int32).view(rows, pages)
    k, v = torch.randn(1 + rows * pages, Hkv, bs, P, generator=g) * 0.8, torch.randn(1 + rows * pages, Hkv, bs, P, generator=g)
    k[0], v[0] = 50.0, 3e4
    for r in range(rows):
        for b in range(pages):
            if held is not None and not held(r, b):
                table[r, b] = 0
    table = torch.cat([table, torch.zeros(1, pages, dtype=torch.int32)]).contiguous()
    return PagedSlot(k.to(dt).to(DEV), v.to(dt).to(DEV), table.to(DEV), bs, None)


@pytest.mark.parametrize("dtype", list(DTYPES))
@pytest.mark.parametrize("chunk,bs", [(1, 4), (5, 4), (16, 16), (24, 16), (40, 16), (64, 16), (100, 4), (333, 16)])
def test_attention_inside_chunks(kernel_sets, dtype, chunk, bs):
    """Decoded tokens, short and long portions that start in the middle of a chunk, pages of earlier chunks given back
    (the null page holds large values), with and without a soft cap, with and without key splits; the first and the last
    token of a chunk among them."""
    ops, dt = kernel_sets[dtype], DTYPES[dtype]
    ref = TorchKernels(dt, DEV)
    g = torch.Generator().manual_seed(chunk * 10 + bs)
    Hkv, P, pages = 2, 32, 448 // bs
    steps = [([200, 1, 1, 37], [0, 3 * chunk % 400, (3 * chunk - 1) % 400, 100]), ([1, 1, 1, 1], [chunk, (2 * chunk - 1) % 400, 0, 399]),
             ([2, 3, 60, 1], [chunk - 1, 2 * chunk % 300 + 1, 7, 5])]
    for G in (1, 4, 3):
        for lengths, starts in steps:
            ctx = _ctx(lengths, [0, 1, 2, 3], starts)
            slot = _paged(dt, Hkv, P, bs, 4, pages, g, held=lambda r, b: (b + 1) * bs > starts[r] // chunk * chunk and b * bs < starts[r] + lengths[r])
            q = torch.randn(ctx.n_tokens, Hkv * G, P, generator=g).to(dt).to(DEV)
            for cap in (None, 5.0):
                terms = {"chunk": chunk, **({"softcap": cap} if cap else {})}
                want = ref.paged_attention(q, slot, ctx, 0.4, None, terms=terms)
                for splits in (None, (112, 4), (16, 28)):
                    ops.attention_splits = splits
                    print("chunked attention", dtype, chunk, bs, G, lengths, cap, splits, flush=True)
                    try:
                        got = ops.paged_attention(q, slot, ctx, 0.4, None, terms=terms)
                    finally:
                        ops.attention_splits = None
                    _close(got, want, dtype, f"chunk {chunk}, {lengths}, cap {cap}, splits {splits}")
    without = ref.paged_attention(q, _paged(dt, Hkv, P, bs, 4, pages, g), ctx, 0.4, None)
    assert not torch.allclose(without.float(), want.float(), atol=0.05)


@pytest.mark.parametrize("row_tiles", [None, 1, 2, 32, 64])
@pytest.mark.parametrize("chunk,P,G", [(40, 32, 2), (100, 64, 1), (64, 128, 4), (7, 48, 2), (500, 64, 3), (33, 32, 1), (1, 16, 4)])
def test_prompt_attention_on_the_matrix_cores_inside_chunks(kernel_sets, chunk, P, G, row_tiles):
    """Long portions through the kernel that shares its key tiles among four or eight waves, in every form, beside single
    tokens and short portions: rows whose block of queries spans a chunk's edge, and blocks inside one chunk."""
    ops, dt = kernel_sets["bfloat16"], torch.bfloat16
    if row_tiles in (32, 64) and P % 32:
        pytest.skip("32-row products take head sizes in steps of 32")
    ref = TorchKernels(dt, DEV)
    g = torch.Generator().manual_seed(chunk + P)
    Hkv, bs = 2, 16
    lengths, starts = [700, 1, 230, 1, 17], [0, 59, 300, 5, 140]
    ctx = _ctx(lengths, [0, 1, 2, 3, 4], starts)
    slot = _paged(dt, Hkv, P, bs, 5, 48, g, held=lambda r, b: (b + 1) * bs > starts[r] // chunk * chunk)
    q = torch.randn(ctx.n_tokens, Hkv * G, P, generator=g).to(dt).to(DEV)
    for cap in (None, 8.0):
        terms = {"chunk": chunk, **({"softcap": cap} if cap else {})}
        want = ref.paged_attention(q, slot, ctx, 0.3, None, terms=terms)
        ops.attention_row_tiles = row_tiles
        print("prompt attention", chunk, P, G, row_tiles, cap, flush=True)
        try:
            got = ops.paged_attention(q, slot, ctx, 0.3, None, terms=terms)
            form = ops.last_attention_kernel
        finally:
            ops.attention_row_tiles = None
        assert row_tiles is None or form == ("workgroup", row_tiles)
        _close(got, want, "bfloat16", f"chunk {chunk}, form {form}, cap {cap}")


def test_chunks_take_the_place_of_a_window(kernel_sets):
    from socrates_amd.kernels import KernelError
    ops = kernel_sets["float32"]
    slot = _paged(torch.float32, 1, 16, 4, 1, 4, torch.Generator().manual_seed(1))
    ctx = _ctx([3], [0], [0])
    q = torch.zeros(3, 1, 16, device=DEV)
    for window, terms in ((4, {"chunk": 4}), (None, {"chunk": 0}), (None, {"chunk": 4, "keep_first": 2})):
        with pytest.raises(KernelError, match="chunk"):
            ops.paged_attention(q, slot, ctx, 1.0, window, terms=terms)


# ---- the models, cut in every way --------------------------------------------------------------------------
def judged_in_bfloat16(got, want, rounded, what):
    """A request in bfloat16 against what rounding alone does to it, which the stand-in kernels in bfloat16 on the CPU
    say (they round where the HIP kernels round): within three times that, by nine rows in ten and by the worst."""
    mine, noise = row_errors(got.cpu(), want), row_errors(rounded, want)
    assert float(mine.max()) <= 3 * float(noise.max()) + 0.02, f"{what}: {float(mine.max()):.3g} against {float(noise.max()):.3g}"
    if mine.numel() >= 10:
        nine = int(0.9 * mine.numel())
        a, b = float(mine.kthvalue(nine).values), float(noise.kthvalue(nine).values)
        assert a <= 3 * b + 0.01, f"{what}, nine rows in ten: {a:.3g} against {b:.3g}"


@pytest.mark.parametrize("dtype", list(DTYPES))
@pytest.mark.parametrize("cut", list(CUTS))
@pytest.mark.parametrize("name", list(MODELS))
def test_cuts_match_the_plain_model(folders, kernel_sets, name, cut, dtype):
    cfg = MODELS[name]
    prompts = random_prompts([3, 41, 70, 26, 1, 58], cfg["vocab"], seed=7)
    pool = dict(num_blocks=4 * (-(-72 // BLOCK[name]))) if cut == "mixed" else {}
    if dtype == "float32":
        check_trace(folders[name, dtype], kernel_sets[dtype], prompts, CUTS[cut](prompts), TOL[dtype], block_size=BLOCK[name], max_len=128,
                    what=f"{name} {cut} {dtype}", graphs=4 if cut in ("tail", "mixed") else 0, **pool)
        return
    runner = make_runner(folders[name, dtype], kernel_sets[dtype], max_rows=4, max_len=128, block_size=BLOCK[name], **pool)
    if cut in ("tail", "mixed"):
        runner.enable_graphs(4)
    got = replay(runner, CUTS[cut](prompts))
    rounded = replay(make_runner(folders[name, dtype], TorchKernels(torch.bfloat16, "cpu"), max_rows=4, max_len=128, block_size=BLOCK[name], **pool),
                     CUTS[cut](prompts))
    want = oracle(folders[name, dtype], prompts)
    for i in range(len(prompts)):
        judged_in_bfloat16(got[f"r{i}"], want[i], rounded[f"r{i}"], f"{name} {cut} request {i}")
    assert runner.cache.open_rows == []


@pytest.mark.parametrize("dtype", list(DTYPES))
@pytest.mark.parametrize("seed", range(24))
def test_drawn_configurations(tmp_path, kernel_sets, seed, dtype):
    """Configurations drawn from everything config.json can say, each under one way of cutting its requests, captured
    decode steps included; in bfloat16 each request is judged against what rounding alone does to it."""
    cfg = drawn_model(seed)
    folder = write_model(tmp_path / "m", cfg, seed=100 + seed, settle=dtype == "bfloat16")
    prompts = random_prompts([23, 1, 40, 9], cfg["vocab"], seed=seed)
    block = [2, 4, 16][seed % 3]
    cut = CUTS[["mixed", "portions", "tail"][seed % 3]]
    runner = make_runner(folder, kernel_sets[dtype], max_rows=4, max_len=40, block_size=block)
    if seed % 2:
        runner.enable_graphs(4)
    got = replay(runner, cut(prompts))
    want = oracle(folder, prompts)
    if dtype == "float32":
        for i in range(len(prompts)):
            compare(got[f"r{i}"], want[i], 1e-3, f"drawn {seed} {dtype} request {i}")
        return
    rounded = replay(make_runner(folder, TorchKernels(torch.bfloat16, "cpu"), max_rows=4, max_len=40, block_size=block), cut(prompts))
    for i in range(len(prompts)):
        judged_in_bfloat16(got[f"r{i}"], want[i], rounded[f"r{i}"], f"drawn {seed} request {i}")


WIDE = model(352, 500, [layer(left(10, 5, 80, 48, 100, scale=0.1), right(6, 2, 72, 104, 4), moe(16, 3, 4, 96)),
                        layer(left(4, 1, 32, 112, 37, scale=0.2), right(5, 5, 96, 40, 3), None, 0.6, 0.9),
                        layer(left(3, 3, 64, 64, 300, scale=0.15), right(4, 1, 136, 32, 2), moe(6, 1, 2, 72), 0.8, -0.7)],
             streams=4, loop=(0, 2, 2), max_positions=768)


@pytest.mark.parametrize("dtype", list(DTYPES))
def test_a_wider_model_with_long_prompts(tmp_path, kernel_sets, dtype):
    """Width 352, heads of 32 to 136, chunks of 37 to 300, prompts of up to 700 tokens: decoded at the end, mixed, and in
    portions of 2 to 200 tokens, through captured decode steps."""
    folder = write_model(tmp_path / "m", WIDE, seed=5, settle=dtype == "bfloat16")
    prompts = random_prompts([700, 333, 64, 150], 500, seed=6)
    want = oracle(folder, prompts)
    for name, steps in (("tail", trace_tail_decode(prompts, 40)), ("mixed", trace_mixed(prompts, seed=7)),
                        ("portions", trace_portions(prompts, seed=8, sizes=(2, 3, 64, 65, 128, 200)))):
        runner = make_runner(folder, kernel_sets[dtype], max_rows=4, max_len=768, block_size=16, num_blocks=4 * 48)
        runner.enable_graphs(4)
        got = replay(runner, steps)
        for i in range(len(prompts)):
            compare(got[f"r{i}"], want[i], TOL[dtype], f"{name} {dtype} request {i}")


@pytest.mark.parametrize("dtype", list(DTYPES))
def test_a_model_of_a_thousand_columns(tmp_path, kernel_sets, dtype):
    """Width 1,024: matrices large enough for the products' other forms (weights read by tile, the sweeps, partial sums,
    the library beyond 16 rows, the experts' large tiles), prompts of up to 300 tokens decoded at the end and mixed."""
    cfg = model(1024, 2000, [layer(left(8, 2, 128, 112, 128, scale=0.06), right(8, 4, 128, 128, 4), moe(7, 1, 2, 512)),
                             layer(left(16, 4, 64, 64, 50, scale=0.1), right(6, 3, 160, 96, 4), moe(3, 2, 2, 768), 0.7, 0.8)], streams=4)
    folder = write_model(tmp_path / "m", cfg, seed=9, settle=dtype == "bfloat16")
    prompts = random_prompts([300, 120, 33], cfg["vocab"], seed=10)
    want = oracle(folder, prompts)
    for name, steps in (("tail", trace_tail_decode(prompts, 24)), ("mixed", trace_mixed(prompts, seed=11))):
        runner = make_runner(folder, kernel_sets[dtype], max_rows=4, max_len=320, block_size=16)
        runner.enable_graphs(4)
        got = replay(runner, steps)
        for i in range(len(prompts)):
            compare(got[f"r{i}"], want[i], TOL[dtype], f"{name} {dtype} request {i}")


@pytest.mark.parametrize("dtype", list(DTYPES))
@pytest.mark.parametrize("chunk", [16, 40])
def test_a_key_just_inside_and_just_outside_the_chunk(tmp_path, kernel_sets, chunk, dtype):
    """One key stands out: the first of the query's chunk, which it sees, and the last of the chunk before, which it does
    not, at the chunk's first tokens and at its end, in a prompt, in portions and decoded from captured steps."""
    cfg = model(56, 60, [layer(left(2, 1, 40, 24, chunk, scale=0.3, softcap=25.0), right(2, 1, 8, 8, 2), None, 1.0, 0.3)], streams=2)
    edge = 2 * chunk
    prompt = random_prompts([edge + chunk + 4], 60, seed=42)[0]
    tol = 3e-4 if dtype == "float32" else 0.05
    for at, seen_from in ((edge, edge + chunk - 1), (edge, edge + chunk), (edge - 1, edge), (edge - 1, edge + 2), (edge, edge + 1)):
        folder = write_model(tmp_path / f"m{at}_{seen_from}", cfg, 41, with_a_sharp_key(cfg, random_weights(cfg, 41), prompt, at, seen_from))
        want = oracle(folder, [prompt])
        if seen_from // chunk != at // chunk:
            other, wd = read_folder(folder)
            other["layers"][0]["mixer"]["left"]["mask"]["size"] = 10 ** 6
            with pytest.raises(AssertionError):
                compare(plain.forward(other, wd, prompt)[seen_from:seen_from + 1], want[0][seen_from:seen_from + 1], 6 * tol)
        for cut in ("whole", "tail", "portions"):
            check_trace(folder, kernel_sets[dtype], [prompt], CUTS[cut]([prompt]), tol, want=want, block_size=8, max_len=edge + chunk + 8,
                        what=f"{at} from {seen_from} {cut}", graphs=1)


@pytest.mark.parametrize("dtype", list(DTYPES))
def test_a_token_far_back_is_carried_by_the_state(tmp_path, kernel_sets, dtype):
    """Token 0 moves the logits 300 places later, through the state alone, whatever the cuts."""
    cfg = model(48, 59, [layer(left(2, 1, 8, 8, 8), right(2, 1, 32, 16, 3), None, 0.5, 1.0)], streams=2)
    w = random_weights(cfg, 6)
    w["l0.mix.right.A_log"] = torch.full((2,), -9.0)
    w["l0.mix.right.b"] = 0.2 * w["l0.mix.right.b"]
    folder = write_model(tmp_path / "m", cfg, 6, w)
    prompt = [58] + [t % 4 for t in random_prompts([304], 59, seed=3)[0]]
    want, moved = oracle(folder, [prompt]), oracle(folder, [[57] + prompt[1:]])
    tol = 3e-4 if dtype == "float32" else 0.03
    far = float(row_errors(moved[0][300:], want[0][300:]).max())
    assert far > 10 * TOL["float32"], far
    for cut in ("whole", "tail", "portions"):
        check_trace(folder, kernel_sets[dtype], [prompt], CUTS[cut]([prompt]), tol, want=want, block_size=16, max_len=320, what=f"state {cut}", graphs=1)


@pytest.mark.parametrize("dtype", list(DTYPES))
def test_long_decoding(folders, kernel_sets, dtype):
    """150 tokens one by one from captured steps, across pages, chunks and context buckets."""
    cfg = MODELS["B"]
    prompts = random_prompts([300], cfg["vocab"], seed=25)
    want = oracle(folders["B", dtype], prompts)
    runner = make_runner(folders["B", dtype], kernel_sets[dtype], max_rows=2, max_len=320, block_size=8)
    runner.enable_graphs(2)
    steps = trace_tail_decode(prompts, 150)
    got = replay(runner, steps)
    if dtype == "float32":
        compare(got["r0"], want[0], TOL[dtype], "decoded")
    else:
        rounded = replay(make_runner(folders["B", dtype], TorchKernels(torch.bfloat16, "cpu"), max_rows=2, max_len=320, block_size=8), steps)
        judged_in_bfloat16(got["r0"], want[0], rounded["r0"], "decoded")


@pytest.mark.parametrize("dtype", list(DTYPES))
def test_captured_decode_steps_equal_eager_ones(folders, kernel_sets, dtype):
    cfg = MODELS["A"]
    prompts = random_prompts([30, 45, 9], cfg["vocab"], seed=31)
    steps = trace_mixed(prompts, seed=32, max_live=3, prefill_frac=0.3)
    eager = replay(make_runner(folders["A", dtype], kernel_sets[dtype], max_len=64, block_size=4), steps)
    runner = make_runner(folders["A", dtype], kernel_sets[dtype], max_len=64, block_size=4)
    runner.enable_graphs(4)
    assert runner.graphs_refused is None and runner.model.capturable
    captured = replay(runner, steps)
    assert runner._graphs, "no decode step was captured"
    tol = 1e-5 if dtype == "float32" else 3e-2          # (a captured step of three rows runs as one of four)
    for rid in eager:
        torch.testing.assert_close(captured[rid], eager[rid], atol=tol * float(eager[rid].std()), rtol=tol)


@pytest.mark.parametrize("name", ["A", "one", "B"])
def test_greedy_generation_through_the_engine(folders, name):
    """``Engine(folder)`` finds the model class by config.json; float32 greedy tokens are the plain model's, with more
    requests than rows, so rows and pages are used again."""
    from socrates_amd.engine import Engine
    cfg, w = read_folder(folders[name, "float32"])
    prompts = random_prompts([5, 17, 33, 2, 21, 11], cfg["vocab"], seed=41)
    want = [plain.greedy(cfg, w, p, 8) for p in prompts]
    engine = Engine(str(folders[name, "float32"]), device=DEV, dtype=torch.float32, max_batch=3, max_len=64, max_new_tokens=8,
                    block_size=BLOCK[name], chunk=16)
    assert engine.generate(prompts, max_new_tokens=8) == want
    engine.cache.check()


def test_command_line(tmp_path, folders):
    """``python -m socrates_amd.generate`` on a model folder, and with ``--random-weights`` on a configuration alone
    (it writes a seeded random model into --model): float32 greedy tokens are the plain model's."""
    cfg, w = read_folder(folders["A", "float32"])
    prompts = random_prompts([5, 17], cfg["vocab"], seed=2)
    want = [plain.greedy(cfg, w, p, 5) for p in prompts]
    cmd = [sys.executable, "-m", "socrates_amd.generate", "--model", str(folders["A", "float32"]), "--dtype", "float32",
           "--max-new-tokens", "5", "--max-len", "64", "--max-batch", "2", "--block-size", "4"]
    for p in prompts:
        cmd += ["--prompt-ids", ",".join(map(str, p))]
    proc = subprocess.run(cmd, capture_output=True, text=True, timeout=300, cwd=str(ROOT))
    assert proc.returncode == 0, proc.stderr[-2000:]
    lines = proc.stdout.strip().split("\n")
    shown = [l for i, l in enumerate(lines) if i > 0 and lines[i - 1].startswith("> ")]
    assert shown == [" ".join(map(str, x)) for x in want]
    (tmp_path / "config.json").write_text(json.dumps(MODELS["B"]))
    made = tmp_path / "made"
    cmd = [sys.executable, "-m", "socrates_amd.generate", "--model", str(made), "--random-weights", str(tmp_path / "config.json"),
           "--seed", "4", "--dtype", "float32", "--max-new-tokens", "4", "--max-len", "64", "--max-batch", "2",
           "--prompt-ids", "7,100,12,5,9"]
    proc = subprocess.run(cmd, capture_output=True, text=True, timeout=300, cwd=str(ROOT))
    assert proc.returncode == 0, proc.stderr[-2000:]
    cfg, w = read_folder(made)
    assert cfg == MODELS["B"]
    lines = proc.stdout.strip().split("\n")
    shown = [l for i, l in enumerate(lines) if i > 0 and lines[i - 1].startswith("> ")]
    assert shown == [" ".join(map(str, plain.greedy(cfg, w, [7, 100, 12, 5, 9], 4)))]


def test_trace_runner_on_a_model_folder(tmp_path, folders):
    cfg = MODELS["A"]
    prompts = random_prompts([70, 33, 100, 12, 64], cfg["vocab"], seed=51)
    steps = trace_mixed(prompts, seed=52)
    lines, wanted, fed = [], [], {}
    for n, (entries, ends) in enumerate(steps):
        lines.append(json.dumps({"step": n, "entries": [{"id": r, "tokens": t, "want": w} for r, t, w in entries], "end": ends}))
        here = []
        for r, t, w in entries:
            here.append((int(r[1:]), [fed.get(r, 0) + j for j in w]))
            fed[r] = fed.get(r, 0) + len(t)
        wanted.append(here)
    max_tokens = sum(-(-len(p) // 64) * 64 for p in sorted(prompts, key=len)[-4:])
    for dtype in DTYPES:
        want = oracle(folders["A", dtype], prompts)
        out = tmp_path / dtype
        proc = subprocess.run([sys.executable, str(ROOT / "bin" / "trace_run"), "--model", str(folders["A", dtype]), "--dtype", dtype,
                               "--out", str(out), "--max-tokens", str(max_tokens)], input="\n".join(lines) + "\n",
                              capture_output=True, text=True, timeout=600)
        assert proc.returncode == 0, proc.stderr[-2000:]
        assert proc.stdout.split("\n")[:-1] == [f"done {i}" for i in range(len(lines))]
        got = {}
        for n, here in enumerate(wanted):
            rows = sum(len(pos) for _, pos in here)
            if rows:
                part = torch.from_numpy(np.fromfile(out / f"{n}.f32", dtype="<f4").reshape(rows, cfg["vocab"]).copy())
                for (i, pos), piece in zip(here, part.split([len(pos) for _, pos in here])):
                    got.setdefault(i, []).append(piece)
        if dtype == "bfloat16":
            rounded = replay(make_runner(folders["A", dtype], TorchKernels(torch.bfloat16, "cpu"), max_rows=4, max_len=128), steps)
        for i in range(len(prompts)):
            if dtype == "float32":
                compare(torch.cat(got[i]), want[i], TOL[dtype], f"request {i} {dtype}")
            else:
                judged_in_bfloat16(torch.cat(got[i]), want[i], rounded[f"r{i}"], f"request {i}")
