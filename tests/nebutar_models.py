"""Small Nebutar configurations and seeded weights for the tests, and the checks that the CPU and the GPU tests share.
Sizes differ from model to model in everything that can differ: head counts of both sides (shared and unshared key heads),
key and value sizes (equal and unequal, none a multiple of 16 among them), chunks shorter and longer than a page and no
multiple of one, one to six taps, one to five copies of the stream, experts from one to fifteen with none to five
identity experts and one to all of them per token, layers without a feed-forward, loops over one layer, over some and
over none, eps, scales of both signs."""

import json
import math
import random
from pathlib import Path

import torch
from safetensors.torch import load_file, save_file

import plain_nebutar as plain
from helpers import make_runner, replay
from mitisun_models import CUTS, compare, row_errors  # noqa: F401  (shared by the test files)


def left(heads, kv_heads, dim, vdim, chunk, scale=None, softcap=20.0):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale or dim ** -0.5, "softcap": softcap,
            "mask": {"size": chunk}}


def right(heads, kv_heads, dim, vdim, conv):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}


def layer(a, b, mlp, left_scale=0.9, right_scale=0.6):
    return {"type": "parallel", "mixer": {"left": a, "right": b, "left_scale": left_scale, "right_scale": right_scale}, "mlp": mlp}


def moe(experts, identity, top, ff):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "identity": identity, "top": top}}


def model(width, vocab, layers, streams, loop=None, eps=1e-5, scale=1.5, max_positions=512):
    cfg = {"architecture": "Nebutar", "vocab": vocab, "width": width, "layers": json.loads(json.dumps(layers)), "norm": {"eps": eps},
           "embedding": {"scale": scale}, "max_positions": max_positions, "streams": streams}
    if loop:
        cfg["loop"] = dict(zip(("start", "stop", "times"), loop))
    return cfg


ONE = model(40, 61, [layer(left(3, 1, 12, 20, 5, scale=0.6), right(4, 2, 12, 20, 3), moe(5, 2, 2, 24))], streams=3)
NO_FFN = model(48, 47, [layer(left(2, 2, 28, 28, 16, softcap=4.0), right(3, 3, 20, 8, 1), None, left_scale=-0.7)] * 2, streams=1, scale=0.7)
FULL = model(36, 53, [layer(left(4, 4, 7, 9, 33), right(2, 1, 9, 33, 6), moe(4, 0, 4, 17), right_scale=-1.1)], streams=2, loop=(0, 1, 3), eps=1e-3)
MIX_A = model(64, 97, [layer(left(4, 2, 16, 24, 24, scale=0.4), right(6, 2, 16, 12, 4), moe(9, 3, 3, 20)),
                       layer(left(6, 1, 32, 16, 7), right(2, 2, 40, 24, 2), None, 0.5, 1.2),
                       layer(left(1, 1, 20, 40, 64, softcap=8.0), right(5, 5, 8, 16, 5), moe(1, 4, 2, 33), -0.6, 0.8),
                       layer(left(3, 3, 44, 12, 1), right(4, 1, 24, 40, 4), moe(15, 1, 5, 12))], streams=4, loop=(1, 3, 2))
MIX_B = model(96, 130, [layer(left(8, 2, 48, 32, 40), right(3, 1, 36, 44, 3), moe(7, 5, 6, 40)),
                        layer(left(5, 5, 24, 48, 100), right(8, 4, 12, 10, 4), moe(3, 2, 1, 64), 1.3, 0.4)], streams=5, loop=(0, 2, 2),
              eps=3e-6, scale=-2.0)
MODELS = {"one": ONE, "no_ffn": NO_FFN, "full": FULL, "A": MIX_A, "B": MIX_B}
BLOCK = {"one": 4, "no_ffn": 8, "full": 16, "A": 4, "B": 16}


def drawn_model(seed):
    """A configuration drawn from everything config.json can say: 1 to 4 layers, sizes that are no multiples of anything
    (and sometimes 1), chunks of one token to more than any prompt, loops or none. (Cached heads come from a short list of
    padded sizes: the attention kernels are compiled per size.)"""
    rng = random.Random(seed)
    width = rng.choice([24, 36, 40, 50, 56, 64, 88, 128])
    layers = []
    for _ in range(rng.randint(1, 4)):
        G, per = rng.choice([1, 1, 2, 3]), rng.choice([1, 1, 2, 4, 5])
        a = left(G * per, G, rng.choice([1, 4, 7, 12, 16, 24, 40]), rng.choice([1, 8, 16, 20, 31, 48, 64]), rng.choice([1, 2, 5, 8, 16, 17, 31, 200]),
                 softcap=rng.choice([1.0, 5.0, 30.0]))
        a["scale"] = rng.choice([0.3, 1.0, 2.0]) * a["dim"] ** -0.5
        G, per = rng.choice([1, 2, 3]), rng.choice([1, 2, 3])
        b = right(G * per, G, rng.choice([1, 3, 4, 12, 16, 31, 64, 70]), rng.choice([1, 5, 8, 16, 17, 40]), rng.randint(1, 6))
        E, same = rng.randint(1, 12), rng.choice([0, 1, 3])
        mlp = None if rng.random() < 0.2 else moe(E, same, rng.randint(1, E + same), rng.choice([8, 24, 50]))
        layers.append(layer(a, b, mlp, rng.choice([-1.0, 0.3, 1.0]), rng.choice([-0.5, 0.7, 1.4])))
    loop = None
    if rng.random() < 0.7:
        start = rng.randrange(len(layers))
        loop = (start, rng.randint(start + 1, len(layers)), rng.randint(1, 3))
    return model(width, rng.choice([37, 64, 101]), layers, streams=rng.choice([1, 2, 3, 4, 6]), loop=loop, eps=rng.choice([1e-6, 1e-5, 1e-3]),
                 scale=rng.choice([0.3, 1.0, 4.0]), max_positions=rng.choice([40, 64, 100]))


def tensor_shapes(cfg):
    d, s = cfg["width"], cfg["streams"]
    t = {"embed": (cfg["vocab"], d), "pos": (cfg["max_positions"], d), "final.norm": (d,), "final.norm.b": (d,)}
    for i, lay in enumerate(cfg["layers"]):
        P, a, b, mlp = f"l{i}.", lay["mixer"]["left"], lay["mixer"]["right"], lay["mlp"]
        for k in ("1", "2") if mlp is not None else ("1",):
            t.update({f"{P}norm{k}": (d,), f"{P}norm{k}.b": (d,), f"{P}hc{k}.in": (s,), f"{P}hc{k}.out": (s,), f"{P}hc{k}.mix": (s, s)})
        p, H, G, D, Dv = P + "mix.left.", a["heads"], a["kv_heads"], a["dim"], a["vdim"]
        t.update({p + "q": (H * D, d), p + "k": (G * D, d), p + "v": (G * Dv, d), p + "o": (d, H * Dv)})
        p, H, G, D, Dv, n = P + "mix.right.", b["heads"], b["kv_heads"], b["dim"], b["vdim"], b["conv"]
        for k, rows in (("q", G * D), ("k", G * D), ("v", H * Dv)):
            t.update({p + k: (rows, d), p + k + ".conv": (rows, n)})
        t.update({p + "b": (H, d), p + "a": (H, d), p + "A_log": (H,), p + "dt_bias": (H,), p + "norm": (Dv,), p + "g": (H * Dv, d),
                  p + "o": (d, H * Dv)})
        if mlp is not None:
            q, E, same, ff = P + "mlp.", mlp["router"]["experts"], mlp["router"]["identity"], mlp["expert"]["ff"]
            t.update({q + "router": (E + same, d), q + "correction": (E + same,)})
            for e in range(E):
                t.update({f"{q}e{e}.gate": (ff, d), f"{q}e{e}.up": (ff, d), f"{q}e{e}.down": (d, ff)})
    return t


def random_weights(cfg, seed):
    """Weights in float32 that already hold bfloat16 values. Matrices are scaled so that every branch has results of order
    one; what reads and writes the copies of the stream differs from copy to copy, decays run from slow to fast, and
    corrections are as large as the scores."""
    g = torch.Generator().manual_seed(seed)
    s = cfg["streams"]
    out = {}
    for name, shape in tensor_shapes(cfg).items():
        r = torch.randn(shape, generator=g)
        leaf = name.split(".")[-1]
        if leaf in ("norm", "norm1", "norm2"):
            t = 1.0 + 0.3 * r
        elif name.endswith((".norm.b", ".norm1.b", ".norm2.b")):
            t = 0.3 * r
        elif leaf == "in":
            t = 1.0 / s + 0.4 * r
        elif leaf == "mix":
            t = 0.8 * torch.eye(s) + 0.3 / math.sqrt(s) * r
        elif leaf == "out":
            t = 1.0 + 0.4 * r
        elif leaf == "A_log":
            t = torch.log(0.02 + 2.0 * torch.rand(shape, generator=g))
        elif leaf == "dt_bias":
            t = -1.0 + r
        elif leaf == "conv":
            t = 0.5 * r
            t[:, -1] += 0.7
        elif leaf == "correction":
            t = 0.15 * r
        elif leaf == "router":
            t = r * (2.0 / math.sqrt(shape[-1]))
        elif name == "embed":
            t = r
        elif name == "pos":
            t = 0.8 * r
        else:
            t = r * (1.5 / math.sqrt(shape[-1]))
        out[name] = t.to(torch.bfloat16).float()
    return out


def settled(w, seed):
    """The same weights with corrections so far apart that no choice of experts hangs on a rounding (scores lie between 0
    and 1): what bfloat16 does to a model whose recurrences would carry one other choice on to every later token."""
    g = torch.Generator().manual_seed(seed)
    return {k: 1.5 * torch.randperm(len(v), generator=g).float() - 2.0 if k.endswith(".correction") else v for k, v in w.items()}


def write_model(folder, cfg, seed, weights=None, settle=False):
    folder = Path(folder)
    folder.mkdir(parents=True, exist_ok=True)
    weights = weights if weights is not None else random_weights(cfg, seed)
    if settle:
        weights = settled(weights, seed)
    (folder / "config.json").write_text(json.dumps(cfg))
    save_file({k: v.to(torch.bfloat16).contiguous() for k, v in weights.items()}, str(folder / "model.safetensors"))
    return folder


def read_folder(folder):
    folder = Path(folder)
    return json.loads((folder / "config.json").read_text()), {k: v.double() for k, v in load_file(str(folder / "model.safetensors")).items()}


_known = {}


def oracle(folder, prompts):
    """The plain model's logits of every prompt (kept: several tests cut the same prompts of one model in their ways)."""
    missing = [p for p in prompts if (str(folder), tuple(p)) not in _known]
    if missing:
        cfg, w = read_folder(folder)
        _known.update({(str(folder), tuple(p)): plain.forward(cfg, w, p).float() for p in missing})
    return [_known[str(folder), tuple(p)] for p in prompts]


def first_inputs(cfg, w, prompt):
    """What layer 0's mixer reads, [T, width] in float64: the normed combination of the embedding output's copies."""
    e = w["embed"].double()[torch.tensor(prompt)] * cfg["embedding"]["scale"] + w["pos"].double()[:len(prompt)]
    return plain.layer_norm(e * w["l0.hc1.in"].double().sum(), w["l0.norm1"].double(), w["l0.norm1.b"].double(), cfg["norm"]["eps"])


def with_a_sharp_key(cfg, w, prompt, at, seen_from, strength=14.0):
    """Weights in which, at layer 0 (its input depends on token and position alone), head 0's query at position
    ``seen_from`` has a capped score of ``strength`` with the key at position ``at`` and of nearly 0 with every other key of
    the prompt (at most as many positions as a key has elements, around the two, are cleared exactly)."""
    w = dict(w)
    m, p = cfg["layers"][0]["mixer"]["left"], "l0.mix.left."
    h, D = first_inputs(cfg, w, prompt), m["dim"]
    keys = h @ w[p + "k"].double()[:D].T
    raw = m["softcap"] * math.atanh(strength / m["softcap"]) / m["scale"]
    lo = max(0, min(at, seen_from) - D // 4)
    some = keys[lo:min(len(prompt), lo + D - 2)] if seen_from - at < D // 2 else torch.cat([keys[lo:lo + D // 2], keys[seen_from - D // 4:seen_from + 1]])
    scores = torch.zeros(len(some), dtype=torch.float64)
    scores[at - lo] = raw
    target = torch.linalg.pinv(some, rcond=1e-3) @ scores
    wq, x = w[p + "q"].double().clone(), h[seen_from]
    wq[:D] += torch.outer(target - wq[:D] @ x, x) / x.dot(x)
    w[p + "q"] = wq.float()
    return w


def check_trace(folder, ops, prompts, steps, tol, want=None, max_rows=4, block_size=16, num_blocks=None, max_len=512, what="", graphs=0):
    """Replay ``steps`` through the framework's step function and compare every position with the oracle."""
    runner = make_runner(folder, ops, max_rows=max_rows, max_len=max_len, block_size=block_size, num_blocks=num_blocks)
    if graphs:
        runner.enable_graphs(graphs)
    got = replay(runner, steps)
    want = want or oracle(folder, prompts)
    for i, p in enumerate(prompts):
        compare(got[f"r{i}"], want[i], tol, f"{what} request {i}")
    assert runner.cache.open_rows == []
    return runner
