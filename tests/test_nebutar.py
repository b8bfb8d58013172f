"""Nebutar through the framework's step function, cache manager and scheduler, on the CPU with the stand-in kernels,
against the plain implementation in ``plain_nebutar``: every mechanism alone and in mixtures; whole prompts,
token-by-token decoding, portions down to two tokens, mixed batches in a pool so small that pages are used again; keys
just inside and just outside a chunk; tokens far back that only the recurrence can carry; looped layers with caches of
their own; the first tokens; long decoding; the configuration and the weights' names."""

import json

import pytest
import torch

import plain_nebutar as plain
from helpers import make_runner, random_prompts, replay, trace_whole
from nebutar_models import (BLOCK, CUTS, MODELS, check_trace, compare, drawn_model, layer, left, model, moe, oracle, random_weights,
                            read_folder, right, tensor_shapes, with_a_sharp_key, write_model)
from socrates_amd.cache import CacheManager
from socrates_amd.config import ConfigError, load_config
from socrates_amd.config.nebutar import NebutarConfig
from socrates_amd.config.specs import LayerNormSpec, RoutedExpertsSpec, StreamsSpec, SwiGLUSpec, WindowAttentionSpec
from socrates_amd.engine import ModelRunner, StepEntry
from socrates_amd.parts import DecoderModel, build_part, cache_needs, expected_tensors
from socrates_amd.parts.registry import PagedKV, RowState
from torch_kernels import TorchKernels

TOL = 2e-4          # float32 stand-in kernels against the float64 oracle, in units of the logits' spread


def ops32():
    return TorchKernels(torch.float32, "cpu")


def ops64():
    return TorchKernels(torch.float64, "cpu", acc=torch.float64)


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    base = tmp_path_factory.mktemp("nebutar")
    return {name: write_model(base / name, cfg, seed=i + 1) for i, (name, cfg) in enumerate(MODELS.items())}


class Steps:
    """Sequences of a step for a kernel that walks them: rows, and where each one's tokens start."""
    def __init__(self, rows, starts):
        self.seq_rows = torch.tensor(rows, dtype=torch.int32)
        self.seq_qstart = torch.tensor(starts, dtype=torch.int32)
        self.n_seqs, self.max_q_len = len(rows), max(b - a for a, b in zip(starts, starts[1:]))


# ---- configuration, plan, names ---------------------------------------------------------------------
def test_plan_follows_the_configuration(folders):
    cfg = load_config(folders["A"])
    assert isinstance(cfg, NebutarConfig) and cfg.to_dict() == MODELS["A"]
    plan = cfg.plan()
    # six runs of four layers; every run has a cache slot of its own, also two passes of one layer
    assert [(s.layer, s.cache, s.write) for s in plan.order] == [(0, 0, True), (1, 1, True), (2, 2, True), (1, 3, True), (2, 4, True), (3, 5, True)]
    needs = cache_needs(plan)
    assert all(isinstance(a, PagedKV) and isinstance(b, RowState) and a.window is None for a, b in needs)
    assert [(a.n_kv_heads, a.head_dim, a.chunk) for a, _ in needs] == [(2, 32, 24), (1, 32, 7), (1, 48, 64), (1, 32, 7), (1, 48, 64), (3, 48, 1)]
    for (_, state), b in zip(needs, [MODELS["A"]["layers"][s.layer]["mixer"]["right"] for s in plan.order]):
        channels = 2 * b["kv_heads"] * b["dim"] + b["heads"] * b["vdim"]
        least = (b["conv"] - 1) * channels + b["heads"] * b["dim"] * b["vdim"]
        assert state.dtype == "float32" and least <= state.shape[0] < least + 8 and state.shape[0] % 4 == 0
    assert plan.head_name is None and plan.streams == 4 and plan.positions_name == "pos" and plan.max_positions == 512
    assert set(plan.ignorable) == {"l1.norm2", "l1.norm2.b", "l1.hc2.in", "l1.hc2.out", "l1.hc2.mix"}
    for name in MODELS:
        names, want = expected_tensors(load_config(folders[name]).plan()), tensor_shapes(MODELS[name])
        assert set(names) == set(want) and all(names[n].fits(want[n]) for n in want), name


def test_configuration_errors():
    def bad(change, match, base="A"):
        cfg = json.loads(json.dumps(MODELS[base]))
        change(cfg)
        with pytest.raises(ConfigError, match=match):
            NebutarConfig.from_dict(cfg)
    bad(lambda c: c.pop("streams"), "streams")
    bad(lambda c: c.update(max_positions=0), "max_positions")
    bad(lambda c: c["norm"].update(eps=0.0), "eps")
    bad(lambda c: c["layers"][0].update(type="attention"), "unknown type")
    bad(lambda c: c["layers"][1]["mixer"].pop("right"), "no sizes")
    bad(lambda c: c["layers"][1]["mixer"]["right"].pop("conv"), "conv")
    bad(lambda c: c["layers"][0]["mixer"]["left"].update(kv_heads=3), "do not divide")
    bad(lambda c: c["layers"][0]["mixer"]["left"].update(scale=-1.0), "scale")
    bad(lambda c: c["layers"][0]["mixer"]["left"].update(softcap=0), "softcap")
    bad(lambda c: c["layers"][0]["mixer"]["left"].update(mask=None), "mask.size")
    bad(lambda c: c["layers"][0]["mixer"].pop("right_scale"), "right_scale")
    bad(lambda c: c["layers"][0]["mlp"].update(kind="dense"), "kind")
    bad(lambda c: c["layers"][0]["mlp"]["router"].update(top=13), "13 of 12")
    bad(lambda c: c["layers"][0]["mlp"]["router"].update(identity=-1), "identity")
    bad(lambda c: c["loop"].update(stop=5), "loop")
    bad(lambda c: c["loop"].update(start=3), "loop")
    bad(lambda c: c["loop"].update(times=0), "loop")
    with pytest.raises(ValueError, match="40 copies"):
        NebutarConfig.from_dict(dict(MODELS["A"], streams=40)).plan()
    # without a loop, and with an identity count left out
    plain_cfg = json.loads(json.dumps(MODELS["A"]))
    plain_cfg.pop("loop")
    plain_cfg["layers"][0]["mlp"]["router"].pop("identity")
    plan = NebutarConfig.from_dict(plain_cfg).plan()
    assert [s.layer for s in plan.order] == [0, 1, 2, 3] and plan.layers[0].ffn.n_identity == 0


def test_spec_errors():
    both = dict(hidden=8, n_heads=2, n_kv_heads=1, head_dim=4, v_dim=4, scale=1.0, eps=1e-5)
    for more in (dict(chunk=0), dict(chunk=4, window=4), dict(chunk=4, keep_first=2)):
        with pytest.raises(ValueError, match="chunk"):
            WindowAttentionSpec(**both, **more)
    with pytest.raises(ValueError, match="identity"):
        RoutedExpertsSpec(hidden=8, n_experts=4, top=1, expert=SwiGLUSpec(8, 8), n_identity=4)
    with pytest.raises(ValueError, match="copies"):
        StreamsSpec(17)


def test_a_layer_without_feed_forward_may_store_what_would_stand_around_it(tmp_path):
    w = random_weights(MODELS["A"], 3)
    w["l1.norm2"], w["l1.norm2.b"], w["l1.hc2.mix"] = torch.ones(64), torch.zeros(64), torch.eye(4)
    make_runner(write_model(tmp_path / "m", MODELS["A"], 3, w), ops32(), max_len=32)


def test_no_row_is_longer_than_the_table_of_positions(tmp_path):
    cfg = dict(MODELS["one"], max_positions=24)
    folder = write_model(tmp_path / "m", cfg, 3)
    with pytest.raises(ValueError, match="24"):
        make_runner(folder, ops32(), max_len=32)
    runner = ModelRunner.from_folder(folder, torch.float32, "cpu", max_rows=2, max_len=64, block_size=4, num_blocks=32, ops=ops32())
    assert runner.cache.max_len == 24
    row = runner.cache.open_row()
    prompt = random_prompts([24], 61, seed=1)[0]
    compare(runner.step([StepEntry(row, prompt, list(range(24)))]), oracle(folder, [prompt])[0], TOL, "up to the last position")
    with pytest.raises(ValueError, match="max_len"):
        runner.step([StepEntry(row, [1], [0])])


# ---- mechanisms alone ---------------------------------------------------------------------------------
@pytest.mark.parametrize("H,G,D,Dv,taps,unit_eps", [(4, 2, 8, 6, 4, 1e-6), (3, 3, 5, 7, 1, 1e-6), (2, 1, 16, 9, 3, 0.1), (6, 2, 1, 1, 6, 1e-6)])
def test_gated_delta_rule_in_portions(H, G, D, Dv, taps, unit_eps):
    """Two sequences' tokens in steps of two and more, beside each other, from states that stay in other rows' places,
    against the plain convolution, unit vectors, gates and walk over the whole."""
    g = torch.Generator().manual_seed(H * 100 + D)
    C, before = 2 * G * D + H * Dv, 3
    conv_len = (taps - 1) * C
    at = (conv_len + 3) // 4 * 4
    state = torch.zeros(3, at + H * D * Dv, dtype=torch.float64)
    w = torch.randn(C, taps, generator=g, dtype=torch.float64)
    a_log, dt = torch.randn(H, generator=g, dtype=torch.float64), torch.randn(H, generator=g, dtype=torch.float64)
    xs = [torch.randn(T, before + C, generator=g, dtype=torch.float64) for T in (19, 11)]
    zs = [torch.randn(T, 2 * H, generator=g, dtype=torch.float64) for T in (19, 11)]
    want = []
    for x, z in zip(xs, zs):
        y = plain.silu(plain.causal_conv(x[:, before:], w))
        q = (plain.unit(y[:, :G * D].view(-1, G, D), unit_eps) * 0.3).repeat_interleave(H // G, 1)
        k = plain.unit(y[:, G * D:2 * G * D].view(-1, G, D), unit_eps).repeat_interleave(H // G, 1)
        gate = torch.exp(-torch.exp(a_log) * torch.log1p(torch.exp(z[:, H:] + dt)))
        o, S = plain.delta_walk(q, k, y[:, 2 * G * D:].view(-1, H, Dv), gate, torch.sigmoid(z[:, :H]))
        want.append((o.reshape(len(x), -1), S))
    got, at_x = [[], []], [0, 0]
    for n0, n1 in ((2, 3), (1, 0), (0, 5), (9, 2), (7, 1)):
        take = [(i, n) for i, n in ((0, n0), (1, n1)) if n]
        ctx = Steps([(2, 0)[i] for i, _ in take], [0] + [sum(n for _, n in take[:k + 1]) for k in range(len(take))])
        cut = lambda t: torch.cat([t[i][at_x[i]:at_x[i] + n] for i, n in take])
        out = ops64().delta_rule(cut(xs), before, G, H, D, Dv, w, 0.3, unit_eps, cut(zs), a_log, dt, state, 0, at, ctx)
        for k, (i, n) in enumerate(take):
            got[i].append(out[ctx.seq_qstart[k]:ctx.seq_qstart[k] + n])
            at_x[i] += n
    for i, row in ((0, 2), (1, 0)):
        torch.testing.assert_close(torch.cat(got[i]), want[i][0], atol=1e-9, rtol=1e-9)
        torch.testing.assert_close(state[row, at:].view(H, Dv, D), want[i][1].transpose(1, 2), atol=1e-9, rtol=1e-9)
    assert not state[1].any()


def test_choice_of_experts_and_identity_experts():
    """Chosen by score + correction, weighted by the score as it is; a choice behind the stacked experts hands its input on."""
    g = torch.Generator().manual_seed(3)
    E, same, d, ff, top = 5, 3, 12, 7, 4
    w = {"router": torch.randn(E + same, d, generator=g, dtype=torch.float64), "correction": 0.3 * torch.randn(E + same, generator=g, dtype=torch.float64)}
    for e in range(E):
        w.update({f"e{e}.gate": torch.randn(ff, d, generator=g, dtype=torch.float64), f"e{e}.up": torch.randn(ff, d, generator=g, dtype=torch.float64),
                  f"e{e}.down": torch.randn(d, ff, generator=g, dtype=torch.float64)})
    x = torch.randn(40, d, generator=g, dtype=torch.float64)
    spec = RoutedExpertsSpec(hidden=d, n_experts=E + same, n_identity=same, top=top, expert=SwiGLUSpec(d, ff, ("gate", "up", "down")), renorm=False)
    part = build_part(spec, w, ops64())
    want = plain.experts_mixture(x, w, "", {"router": {"experts": E, "identity": same, "top": top}})
    # (router logits are float32 in every kernel set)
    torch.testing.assert_close(part.forward(x)[0], want, atol=1e-5, rtol=1e-5)
    torch.testing.assert_close(part.forward(x, whole=False), want, atol=1e-5, rtol=1e-5)
    chosen, weights = plain.router(x, w, "", top)
    assert bool((chosen >= E).any()) and bool((chosen < E).any()) and bool((weights.sum(-1) < 0.999).any())


def test_layer_norm_is_a_norm_like_the_others():
    """The norm with mean and bias as a part of its own: on a plain stream, with and without a sum to add, and on
    selected rows."""
    g = torch.Generator().manual_seed(4)
    w, b = torch.randn(9, generator=g), torch.randn(9, generator=g)
    norm = build_part(LayerNormSpec(9, 1e-3), {"": w, "b": b}, ops32())
    x, y = torch.randn(6, 9, generator=g), torch.randn(6, 9, generator=g)
    stream = x.clone()
    torch.testing.assert_close(norm.add_norm(stream, None), plain.layer_norm(x, w, b, 1e-3))
    rows = torch.tensor([4, 1], dtype=torch.int32)
    torch.testing.assert_close(norm.add_norm(stream, y, rows), plain.layer_norm((x + y)[[4, 1]], w, b, 1e-3))
    assert torch.equal(stream, x)
    torch.testing.assert_close(norm.add_norm(stream, y), plain.layer_norm(x + y, w, b, 1e-3))
    torch.testing.assert_close(stream, x + y)


def test_copies_of_the_stream():
    """All copies at once from the old ones, the mix indexed [from, to], against the plain function."""
    g = torch.Generator().manual_seed(5)
    s, T, d = 3, 7, 8
    x, y = torch.randn(s, T, d, generator=g), torch.randn(T, d, generator=g)
    w = {"in": torch.randn(s, generator=g), "mix": torch.randn(s, s, generator=g), "out": torch.randn(s, generator=g)}
    want = plain.through_streams(x, w, "", lambda u: y)
    mine = x.transpose(0, 1).contiguous()
    ops32().streams_update(mine, [(0.5 * y, 2.0)], w["mix"], w["out"])
    torch.testing.assert_close(mine.transpose(0, 1), want)
    assert float((want - plain.through_streams(x, dict(w, mix=w["mix"].T), "", lambda u: y)).abs().max()) > 0.1


def test_every_mechanism_shows(folders):
    """The plain model with one constant changed differs from the framework by far more than the tolerance: what the
    other tests compare would not hide such a fault."""
    for name in ("A", "B"):
        cfg, w = read_folder(folders[name])
        prompt = random_prompts([60], cfg["vocab"], seed=13)[0]
        check_trace(folders[name], ops32(), [prompt], CUTS["portions"]([prompt]), TOL, max_len=64, what=name)
        want = plain.forward(cfg, w, prompt)

        def with_sides(**change):
            other = json.loads(json.dumps(cfg))
            for lay in other["layers"]:
                for side, keys in change.items():
                    for k, f in keys.items():
                        lay["mixer"][side][k] = f(lay["mixer"][side][k])
            return other

        def with_weights(match, f):
            return {k: f(v) if k.endswith(match) else v for k, v in w.items()}
        changes = {"a longer chunk": (with_sides(left={"mask": lambda m: {"size": m["size"] + 1}}), w),
                   "another soft cap": (with_sides(left={"softcap": lambda c: 0.6 * c}), w),
                   "no correction": (cfg, with_weights(".correction", torch.zeros_like)),
                   "no norm bias": (cfg, with_weights((".norm1.b", ".norm2.b"), torch.zeros_like)),
                   "one pass fewer": (dict(cfg, loop=dict(cfg["loop"], times=1)), w),
                   "no positions": (cfg, with_weights("pos", torch.zeros_like)),
                   "taps the other way round": (cfg, with_weights(".conv", lambda v: v.flip(1))),
                   "another decay": (cfg, with_weights(".A_log", lambda v: v + 0.7)),
                   "another step": (cfg, with_weights(".dt_bias", lambda v: v + 1.0)),
                   "mix turned round": (cfg, with_weights(".mix", lambda v: v.T.contiguous())),
                   "head norms without a gain": (cfg, with_weights(".mix.right.norm", torch.ones_like)),
                   "unscaled embedding": (dict(cfg, embedding={"scale": 1.0}), w)}
        if cfg["norm"]["eps"] > 1e-4:
            changes["eps"] = (dict(cfg, norm={"eps": 1e-8}), w)
        for what, (cc, ww) in changes.items():
            with pytest.raises(AssertionError):
                compare(plain.forward(cc, ww, prompt), want, 20 * TOL, what)
                print(f"{name}: {what} does not show")


# ---- the models, cut in every way ------------------------------------------------------------------------
@pytest.mark.parametrize("cut", list(CUTS))
@pytest.mark.parametrize("name", list(MODELS))
def test_cuts_match_the_plain_model(folders, name, cut):
    cfg = MODELS[name]
    prompts = random_prompts([3, 41, 70, 26, 1, 58], cfg["vocab"], seed=7)
    # a pool that cannot hold all requests at once: pages come back and are used again
    pool = dict(num_blocks=4 * (-(-72 // BLOCK[name]))) if cut == "mixed" else {}
    check_trace(folders[name], ops32(), prompts, CUTS[cut](prompts), TOL, block_size=BLOCK[name], max_len=128, what=f"{name} {cut}", **pool)


def test_a_batch_equals_each_request_alone(folders):
    cfg = MODELS["A"]
    prompts = random_prompts([37, 2, 19, 64], cfg["vocab"], seed=9)
    runner = make_runner(folders["A"], ops32(), max_len=128)
    alone = []
    for p in prompts:
        row = runner.cache.open_row()
        alone.append(runner.step([StepEntry(row, p, list(range(len(p))))]))
        runner.cache.close_row(row)
    rows = [runner.cache.open_row() for _ in prompts]
    together = runner.step([StepEntry(r, p, list(range(len(p)))) for r, p in zip(rows, prompts)])
    compare(together, torch.cat(alone), 1e-5, "batch against alone")


def test_passes_of_a_looped_layer_keep_caches_and_states_of_their_own(folders):
    """After a prompt the slots of two passes of one layer hold different keys and states, and a request taken up again
    much later, with others in between, goes on from its own."""
    cfg = MODELS["A"]
    prompts = random_prompts([33, 20, 25], cfg["vocab"], seed=10)
    runner = make_runner(folders["A"], ops32(), max_rows=3, max_len=64, block_size=4)
    want = oracle(folders["A"], prompts)
    rows = [runner.cache.open_row() for _ in prompts]
    runner.step([StepEntry(rows[0], prompts[0][:17], [])])
    (a, sa), (b, sb) = runner.cache.slot(2), runner.cache.slot(4)
    pages = a.block_table[rows[0], :4].long()
    assert a.k.data_ptr() != b.k.data_ptr() and float((a.k[pages] - b.k[pages]).abs().max()) > 0.1
    assert float((sa.state[rows[0]] - sb.state[rows[0]]).abs().max()) > 0.1
    for r, p, n in ((1, prompts[1], 1), (2, prompts[2], 2)):
        got = runner.step([StepEntry(rows[r], p, list(range(len(p))))])
        compare(got, want[n], TOL, f"request {n}")
    got = runner.step([StepEntry(rows[0], prompts[0][17:], list(range(16)))])
    compare(got, want[0][17:], TOL, "taken up again")


def test_rows_and_pages_used_again_start_clean(folders):
    cfg = MODELS["B"]
    a, b = random_prompts([50, 33], cfg["vocab"], seed=11)
    runner = make_runner(folders["B"], ops32(), max_rows=1, max_len=64, block_size=4, num_blocks=16)
    want = oracle(folders["B"], [b])[0]
    for first in (a, b, a):
        row = runner.cache.open_row()
        runner.step([StepEntry(row, first, [])])
        runner.cache.close_row(row)
    row = runner.cache.open_row()
    assert row == 0
    got = torch.cat([runner.step([StepEntry(row, b[:20], list(range(20)))]), runner.step([StepEntry(row, b[20:], list(range(13)))])])
    compare(got, want, TOL, "pages used again")


@pytest.mark.parametrize("chunk,block", [(8, 4), (24, 16), (5, 4), (1, 2), (3, 8)])
def test_pages_of_earlier_chunks_come_back(chunk, block):
    """A page all of whose positions lie in chunks before the next token's is given back, no other one is."""
    cache = CacheManager([PagedKV(1, 16, chunk=chunk)], max_rows=2, max_len=128, block_size=block, num_blocks=64, dtype=torch.float32, device="cpu")
    row, n = cache.open_row(), 0
    rest = [7, 1, 1, 9, 2, 1, 13, 1, 1, 20, 1, 8, 1, 1, 1, 30]
    for step in rest:
        cache.reserve(row, n + step)
        first = n // chunk * chunk                                    # the first position the step's first token sees
        held = {b for b in range(-(-(n + step) // block)) if (b + 1) * block > first}
        assert {int(b) for b in cache.groups[0].host_table[row].nonzero()[0]} == held, n
        cache.advance(row, step)
        n += step
        cache.check()
    cache.close_row(row)
    cache.check()
    assert cache.groups[0].allocator.n_free == 64


def test_chunks_and_windows_do_not_mix():
    for need in (PagedKV(1, 16, window=4, chunk=4), PagedKV(1, 16, chunk=0), PagedKV(1, 16, keep_first=2, chunk=4)):
        with pytest.raises(ValueError, match="chunk"):
            CacheManager([need], max_rows=1, max_len=32, block_size=4, num_blocks=8, dtype=torch.float32, device="cpu")


@pytest.mark.parametrize("chunk", [16, 24, 33])
def test_a_key_just_inside_and_just_outside_the_chunk(tmp_path, chunk):
    """One key stands out: the first of the query's chunk, which it sees, and the last of the chunk before, which it does
    not (a chunk one token longer or shorter would), at the chunk's first tokens and at its end, in prompts and decoded."""
    base = model(56, 60, [layer(left(2, 1, 40, 24, chunk, scale=0.3, softcap=25.0), right(2, 1, 8, 8, 2), None, 1.0, 0.3)], streams=2)
    edge = 2 * chunk
    prompt = random_prompts([edge + chunk + 4], 60, seed=42)[0]
    cases = [(edge, edge + chunk - 1, True), (edge, edge + chunk, False), (edge - 1, edge, False), (edge - 1, edge + 2, False), (edge, edge + 1, True)]
    for at, seen_from, inside in cases:
        w = with_a_sharp_key(base, random_weights(base, 41), prompt, at, seen_from)
        folder = write_model(tmp_path / f"m{at}_{seen_from}", base, 41, w)
        want = oracle(folder, [prompt])
        cfg, wd = read_folder(folder)
        # where the key lies outside, a model without chunks would look at it
        other = json.loads(json.dumps(cfg))
        other["layers"][0]["mixer"]["left"]["mask"]["size"] = 10 ** 6
        unmasked = plain.forward(other, wd, prompt)[seen_from]
        if not inside:
            with pytest.raises(AssertionError):
                compare(unmasked.unsqueeze(0), want[0][seen_from:seen_from + 1].double(), 100 * TOL)
        moved = list(prompt)
        moved[at] = (prompt[at] + 1) % 60
        changed = oracle(folder, [moved])[0]
        shift = (changed[seen_from] - want[0][seen_from]).abs().max() / want[0][seen_from].std()
        assert float(shift) > (100 * TOL if inside else 0), (at, seen_from)
        for cut in ("whole", "tail", "portions"):
            check_trace(folder, ops32(), [prompt], CUTS[cut]([prompt]), TOL, want=want, block_size=8, max_len=edge + chunk + 8,
                        what=f"{at} from {seen_from}, {cut}")


def slow_model(seed):
    """A model in which nothing but the recurrence reaches far back: chunks of 8, decays near one and small steps."""
    cfg = model(48, 59, [layer(left(2, 1, 8, 8, 8), right(2, 1, 32, 16, 3), None, 0.5, 1.0)], streams=2)
    w = random_weights(cfg, seed)
    w["l0.mix.right.A_log"] = torch.full((2,), -9.0)
    w["l0.mix.right.b"] = 0.2 * w["l0.mix.right.b"]
    return cfg, w


def test_a_token_far_back_is_carried_by_the_state(tmp_path):
    """Token 0 moves the logits 200 places later, through the state alone, whatever the cuts."""
    cfg, w = slow_model(6)
    folder = write_model(tmp_path / "m", cfg, 6, w)
    prompt = random_prompts([205], 59, seed=3)[0]
    # a vocabulary of few tokens fills the state over and over: the later tokens are drawn from a handful
    prompt = [58] + [t % 4 for t in prompt[1:]]
    want = oracle(folder, [prompt])
    moved = oracle(folder, [[57] + prompt[1:]])
    with pytest.raises(AssertionError):
        compare(moved[0][200:], want[0][200:], 10 * TOL)
    for cut in ("whole", "tail", "portions"):
        check_trace(folder, ops32(), [prompt], CUTS[cut]([prompt]), TOL, want=want, block_size=16, max_len=208, what=f"state {cut}")


def test_the_first_tokens(folders):
    """Single tokens from the very start: convolutions before which nothing lies, empty states, first positions."""
    for name in MODELS:
        prompts = random_prompts([7, 1, 2], MODELS[name]["vocab"], seed=6)
        steps = [([(f"r{i}", [t], [0])], [f"r{i}"] if n + 1 == len(p) else []) for i, p in enumerate(prompts) for n, t in enumerate(p)]
        check_trace(folders[name], ops32(), prompts, steps, TOL, max_len=16, what=f"{name} first tokens")


@pytest.mark.parametrize("seed", range(12))
def test_drawn_configurations(tmp_path, seed):
    cfg = drawn_model(seed)
    folder = write_model(tmp_path / "m", cfg, seed=100 + seed)
    prompts = random_prompts([23, 1, 40, 9], cfg["vocab"], seed=seed)
    block = [2, 4, 16][seed % 3]
    # (such models can be touchy in float32: a sharp softmax, a width of 24; a fault is larger by far)
    check_trace(folder, ops32(), prompts, CUTS[["mixed", "portions", "tail"][seed % 3]](prompts), 5 * TOL, block_size=block,
                max_len=40, what=f"drawn {seed}")


def test_long_decoding(folders):
    cfg = MODELS["one"]
    prompts = random_prompts([230], cfg["vocab"], seed=25)
    steps = [([("r0", prompts[0][:5], list(range(5)))], [])]
    steps += [([("r0", [t], [0])], []) for t in prompts[0][5:]]
    steps[-1] = (steps[-1][0], ["r0"])
    check_trace(folders["one"], ops32(), prompts, steps, TOL, max_len=256, what="225 decoded tokens")


def test_greedy_generation_through_the_engine(folders):
    """The framework's own entry point and scheduler over this model: more requests than rows, prompts cut into portions,
    rows used again; the tokens are the plain model's greedy ones."""
    from socrates_amd.engine import Engine
    cfg, w = read_folder(folders["A"])
    prompts = random_prompts([12, 3, 29, 7, 18], cfg["vocab"], seed=26)
    want = [plain.greedy(cfg, w, p, 6) for p in prompts]
    runner = make_runner(folders["A"], ops64(), max_rows=3, max_len=64, block_size=4)
    engine = Engine(runner, device="cpu", dtype=torch.float64, compile=False, max_batch=3, max_len=64, max_new_tokens=6,
                    block_size=4, chunk=8)
    assert engine.generate(prompts, max_new_tokens=6) == want


def test_tokens_do_not_depend_on_the_pool(folders):
    """Pools so small that requests wait and have their portions shortened, or are preempted and computed again: float64
    greedy tokens are those of a roomy pool and of the plain model."""
    from socrates_amd.engine import Engine
    cfg, w = read_folder(folders["B"])
    prompts = random_prompts([5, 17, 33, 9, 24, 40, 1, 12], cfg["vocab"], seed=27)
    want = [plain.greedy(cfg, w, p, 8) for p in prompts]
    for num_blocks, chunk in ((64, 2048), (14, 7), (13, 5)):
        runner = make_runner(folders["B"], ops64(), max_rows=4, max_len=64, block_size=4, num_blocks=num_blocks)
        engine = Engine(runner, device="cpu", dtype=torch.float64, compile=False, max_batch=4, max_len=64, max_new_tokens=8,
                        block_size=4, chunk=chunk)
        assert engine.generate(prompts, max_new_tokens=8) == want, (num_blocks, chunk)
        engine.cache.check()
        assert not engine.cache.open_rows and all(g.allocator.n_free == g.allocator.num_blocks for g in engine.cache.groups)
    with pytest.raises(Exception, match="exceeds"):
        engine.submit(list(range(60)))


def test_one_copy_with_plain_weights_is_a_prenorm_layer(tmp_path):
    """With one copy of the stream read, kept and written with weight one, the model is the pre-norm one."""
    cfg = MODELS["no_ffn"]
    w = random_weights(cfg, 2)
    for k in w:
        if ".hc" in k:
            w[k] = torch.ones_like(w[k])
    folder = write_model(tmp_path / "m", cfg, 2, w)
    prompt = random_prompts([30], cfg["vocab"], seed=4)[0]
    wd = {k: v.double() for k, v in w.items()}
    x = wd["embed"][torch.tensor(prompt)] * cfg["embedding"]["scale"] + wd["pos"][:30]
    for i in (0, 1):
        h = plain.layer_norm(x, wd[f"l{i}.norm1"], wd[f"l{i}.norm1.b"], 1e-5)
        x = x + plain.parallel_mixer(h, wd, f"l{i}.mix.", cfg["layers"][i]["mixer"], 1e-5)
    want = plain.layer_norm(x, wd["final.norm"], wd["final.norm.b"], 1e-5) @ wd["embed"].T
    got = replay(make_runner(folder, ops32(), max_len=32), trace_whole([prompt]))["r0"]
    compare(got, want, TOL, "prenorm")


def test_the_mixer_sums_its_sides_itself_where_no_block_does(folders):
    """The parallel mixer in a block that takes one result: the same sum as where the block adds the sides up."""
    cfg, w = read_folder(folders["A"])
    plan = load_config(folders["A"]).plan()
    ops = ops64()
    model = DecoderModel(plan, {k: v.clone() for k, v in w.items()}, ops)
    x = torch.randn(9, 64, generator=torch.Generator().manual_seed(1), dtype=torch.float64)
    for k in (0, 1):
        spec = plan.layers[k].mixer
        mixer = model.blocks[k].mixer
        out = []
        for apart in (False, True):
            cache = CacheManager([cache_needs(plan)[k]], max_rows=1, max_len=16, block_size=4, num_blocks=4, dtype=torch.float64, device="cpu")
            row = cache.open_row()
            cache.reserve(row, 9)
            from socrates_amd.engine.batch import build_context
            ctx = build_context([StepEntry(row, [0] * 9, [])], [0], "cpu")
            y = mixer.forward(x, ctx, cache.slot(0), apart=apart)
            out.append((y if not apart else sum(s * t for t, s in y)).double())
        torch.testing.assert_close(out[0], out[1], atol=1e-5, rtol=1e-5)
        assert spec.left_scale != 1.0
