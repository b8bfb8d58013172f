"""Typed configuration of Nebutar (``"architecture": "Nebutar"``).

A decoder whose layers keep two mixers side by side on one input (``layers`` lists them, ``type`` "parallel"): grouped-query
softmax attention inside fixed chunks of positions, without positions in the scores and with a soft cap on them, beside the
gated delta rule with short convolutions; the two results are scaled and added. Feed-forwards are mixtures of silu-gated
experts chosen by corrected softmax scores and weighted by the scores themselves, the last outputs of the router standing
for experts that hand their input on (or a layer has none). The residual stream is kept in ``streams`` copies that every
branch reads and writes through stored weights; norms take the mean off and have a bias; learned positions are added to
the scaled embedding. ``loop`` runs layers start .. stop - 1 several times in a row, each pass with a cache and state of
its own. Tensor names: layer i's start with ``l<i>.``, the mixer's with ``l<i>.mix.left.`` and ``l<i>.mix.right.``, the
feed-forward's with ``l<i>.mlp.``, the copies' weights with ``l<i>.hc1.`` and ``l<i>.hc2.``; the output head is the embedding
table.
"""

from __future__ import annotations

import json
from dataclasses import dataclass
from pathlib import Path
from typing import Optional, Tuple

from .mitisun import _freeze, _positive_int, _thaw
from .qwen3 import ConfigError
from .specs import (BlockSpec, GatedDeltaSpec, LayerNormSpec, ModelPlan, ParallelMixerSpec, RoutedExpertsSpec, RunStep, StreamsSpec,
                    SwiGLUSpec, WindowAttentionSpec)
from .tedulorn import _number

_NAMES = (("norm1", "norm1"), ("mixer", "mix"), ("norm2", "norm2"), ("ffn", "mlp"), ("streams1", "hc1"), ("streams2", "hc2"))
_LEFT_KEYS = ("heads", "kv_heads", "dim", "vdim")
_RIGHT_KEYS = ("heads", "kv_heads", "dim", "vdim", "conv")


def _sizes(where, m, keys):
    if not isinstance(m, dict):
        raise ConfigError(f"{where}: no sizes")
    lacking = [k for k in keys if k not in m]
    if lacking:
        raise ConfigError(f"{where} lacks {lacking}")
    for k in keys:
        _positive_int(where, k, m[k])
    if m["heads"] % m["kv_heads"]:
        raise ConfigError(f"{where}: {m['heads']} heads do not divide into {m['kv_heads']} kv heads")


def _whole(where, key, value):
    if not isinstance(value, int) or isinstance(value, bool) or value < 0:
        raise ConfigError(f"{where}: {key} must be a whole number, not negative, found {value!r}")
    return value


@dataclass(frozen=True)
class NebutarConfig:
    vocab: int
    width: int
    layers: Tuple[tuple, ...]         # as config.json lists them (validated, frozen)
    norm_eps: float
    embedding_scale: float
    max_positions: int
    streams: int
    loop: Optional[Tuple[int, int, int]] = None      # (start, stop, times)
    eos_token_ids: Tuple[int, ...] = ()
    architecture: str = "Nebutar"

    # ---- reading -----------------------------------------------------------------
    @classmethod
    def from_dict(cls, d: dict) -> "NebutarConfig":
        missing = [k for k in ("vocab", "width", "layers", "norm", "max_positions", "streams") if k not in d]
        if missing:
            raise ConfigError(f"config.json lacks {missing} (required for Nebutar)")
        for k in ("vocab", "width", "max_positions", "streams"):
            _positive_int("config", k, d[k])
        if not isinstance(d["norm"], dict) or not d["norm"].get("eps", 0) > 0:
            raise ConfigError("norm.eps must be positive")
        scale = 1.0
        if d.get("embedding") is not None:
            scale = _number("config", "embedding.scale", (d["embedding"] or {}).get("scale", 1.0), positive=False)
        if not isinstance(d["layers"], (list, tuple)) or not d["layers"]:
            raise ConfigError("layers must list at least one layer")
        layers = []
        for i, layer in enumerate(d["layers"]):
            where = f"layer {i}"
            if layer.get("type") != "parallel":
                raise ConfigError(f"{where}: unknown type {layer.get('type')!r}; known: ['parallel']")
            m = layer.get("mixer")
            if not isinstance(m, dict):
                raise ConfigError(f"{where}: no mixer sizes")
            left, right = m.get("left"), m.get("right")
            _sizes(f"{where}, left", left, _LEFT_KEYS)
            _sizes(f"{where}, right", right, _RIGHT_KEYS)
            _number(f"{where}, left", "scale", left.get("scale"))
            _number(f"{where}, left", "softcap", left.get("softcap"))
            _positive_int(f"{where}, left", "mask.size", (left.get("mask") or {}).get("size"))
            for k in ("left_scale", "right_scale"):
                _number(where, k, m.get(k), positive=False)
            mlp = layer.get("mlp")
            if mlp is not None:
                if mlp.get("kind") != "moe":
                    raise ConfigError(f"{where}: feed-forward kind {mlp.get('kind')!r} is not known (moe)")
                _positive_int(where, "mlp.expert.ff", (mlp.get("expert") or {}).get("ff"))
                r = mlp.get("router")
                if not isinstance(r, dict):
                    raise ConfigError(f"{where}: mlp.router is missing")
                E = _positive_int(where, "router.experts", r.get("experts"))
                same = _whole(where, "router.identity", r.get("identity", 0))
                if _positive_int(where, "router.top", r.get("top")) > E + same:
                    raise ConfigError(f"{where}: {r['top']} of {E + same} experts is not possible")
            layers.append(json.loads(json.dumps(layer)))       # a copy of plain values
        loop = None
        if d.get("loop") is not None:
            if not isinstance(d["loop"], dict):
                raise ConfigError("loop needs start, stop and times")
            start, stop, times = (_whole("loop", k, d["loop"].get(k)) for k in ("start", "stop", "times"))
            if not start < stop <= len(layers) or times < 1:
                raise ConfigError(f"loop: layers {start} .. {stop} of {len(layers)}, {times} times")
            loop = (start, stop, times)
        eos = d.get("eos_token_id")
        eos_ids = () if eos is None else tuple(eos) if isinstance(eos, (list, tuple)) else (int(eos),)
        return cls(vocab=d["vocab"], width=d["width"], layers=tuple(_freeze(x) for x in layers), norm_eps=float(d["norm"]["eps"]),
                   embedding_scale=scale, max_positions=d["max_positions"], streams=d["streams"], loop=loop, eos_token_ids=eos_ids,
                   architecture=d.get("architecture", "Nebutar"))

    @classmethod
    def from_json(cls, path) -> "NebutarConfig":
        path = Path(path)
        if path.is_dir():
            path = path / "config.json"
        return cls.from_dict(json.loads(path.read_text()))

    # ---- writing -----------------------------------------------------------------
    def to_dict(self) -> dict:
        out = {"architecture": self.architecture, "embedding": {"scale": self.embedding_scale},
               "layers": [_thaw(x) for x in self.layers], "max_positions": self.max_positions, "norm": {"eps": self.norm_eps},
               "streams": self.streams, "vocab": self.vocab, "width": self.width}
        if self.loop is not None:
            out["loop"] = dict(zip(("start", "stop", "times"), self.loop))
        if self.eos_token_ids:
            out["eos_token_id"] = self.eos_token_ids[0] if len(self.eos_token_ids) == 1 else list(self.eos_token_ids)
        return out

    # ---- the layer recipe -------------------------------------------------------------
    def _mixer(self, m):
        d, eps = self.width, self.norm_eps
        left, right = m["left"], m["right"]
        return ParallelMixerSpec(
            left=WindowAttentionSpec(hidden=d, n_heads=left["heads"], n_kv_heads=left["kv_heads"], head_dim=left["dim"],
                                     v_dim=left["vdim"], scale=float(left["scale"]), eps=eps, softcap=float(left["softcap"]),
                                     chunk=left["mask"]["size"]),
            right=GatedDeltaSpec(hidden=d, n_heads=right["heads"], n_kv_heads=right["kv_heads"], head_dim=right["dim"],
                                 v_dim=right["vdim"], conv_taps=right["conv"], eps=eps),
            left_scale=float(m["left_scale"]), right_scale=float(m["right_scale"]))

    def _ffn(self, mlp):
        d = self.width
        if mlp is None:
            return None
        r = mlp["router"]
        same = r.get("identity", 0)
        return RoutedExpertsSpec(hidden=d, n_experts=r["experts"] + same, n_identity=same, top=r["top"],
                                 expert=SwiGLUSpec(d, mlp["expert"]["ff"], ("gate", "up", "down")), renorm=False)

    def run_layers(self):
        """The layers in the order they run, a looped one as often as it runs."""
        n = len(self.layers)
        if self.loop is None:
            return list(range(n))
        start, stop, times = self.loop
        return list(range(start)) + list(range(start, stop)) * times + list(range(stop, n))

    def plan(self) -> ModelPlan:
        d = self.width
        norm, copies = LayerNormSpec(d, self.norm_eps), StreamsSpec(self.streams)
        blocks, ignorable = [], []
        for i, layer in enumerate(_thaw(x) for x in self.layers):
            ffn = self._ffn(layer.get("mlp"))
            if ffn is None:                 # (a file may hold what would stand around a feed-forward that the layer lacks)
                ignorable += [f"l{i}.norm2", f"l{i}.norm2.b"] + [f"l{i}.hc2.{k}" for k in ("in", "out", "mix")]
            blocks.append(BlockSpec(mixer=self._mixer(layer["mixer"]), ffn=ffn, norm1=norm, norm2=None if ffn is None else norm,
                                    prefix=f"l{i}.", names=_NAMES, arrangement="streams", streams1=copies,
                                    streams2=None if ffn is None else copies))
        # every pass of a looped layer runs the same block with a cache slot of its own
        order = tuple(RunStep(layer=i, cache=k) for k, i in enumerate(self.run_layers()))
        return ModelPlan(
            architecture=self.architecture, vocab_size=self.vocab, hidden=d, layers=tuple(blocks), order=order, final_norm=norm,
            embedding_name="embed", final_norm_prefix="final.norm", head_name=None, eos_token_ids=self.eos_token_ids,
            ignorable=tuple(ignorable), embedding_scale=self.embedding_scale, positions_name="pos",
            max_positions=self.max_positions, streams=self.streams)

    # ---- byte and flop counts ---------------------------------------------------------
    def _weighted_elements(self, plan, share_of):
        """Stored matrix elements of the layers, as often as each runs, an expert's times ``share_of`` its feed-forward."""
        from ..parts import expected_tensors
        times = [sum(step.layer == k for step in plan.order) for k in range(len(plan.layers))]
        total = 0.0
        for name, decl in expected_tensors(plan).items():
            if name in ("embed", "pos") or decl.kind != "matrix":
                continue
            k = next(k for k, block in enumerate(plan.layers) if name.startswith(block.prefix))
            n = decl.shape[0] * decl.shape[1] * times[k]
            if name.startswith(plan.layers[k].prefix + "mlp.e"):
                n *= share_of(plan.layers[k].ffn)
            total += n
        return total

    def step_weight_bytes(self, batch: int, item: int) -> int:
        """Bytes of weights that a decode step of ``batch`` tokens reads if its tokens choose their experts independently
        and evenly (of E outputs of the router, each is chosen with 1 - (1 - top / E)^batch); a layer is read as often
        as it runs; the head is the embedding table, read whole."""
        body = self._weighted_elements(self.plan(), lambda f: 1.0 - (1.0 - f.top / f.n_experts) ** batch)
        return int((body + self.vocab * self.width) * item)

    def step_cache_bytes(self, batch: int, context: int, item: int) -> int:
        """Bytes of cache and state that a decode step of ``batch`` requests behind ``context`` tokens reads and, of the
        matrix states, writes."""
        plan = self.plan()
        total = 0
        for step in plan.order:
            left, right = plan.layers[step.layer].mixer.left, plan.layers[step.layer].mixer.right
            total += 2 * 4 * right.n_heads * right.head_dim * right.v_dim
            total += item * 2 * left.n_kv_heads * left.cache_width * (context % left.chunk + 1)
        return batch * total

    def prefill_flops(self, tokens: int) -> float:
        """Multiply-adds times two of one prompt of ``tokens`` tokens from position 0: every matrix a token uses (of the
        experts a token's share; the head at one position), attention inside the chunks, and the recurrence (per
        token and head, state size times six)."""
        plan = self.plan()
        flops = 2.0 * tokens * self._weighted_elements(plan, lambda f: f.top / f.n_experts) + 2.0 * self.vocab * self.width
        for step in plan.order:
            left, right = plan.layers[step.layer].mixer.left, plan.layers[step.layer].mixer.right
            c = left.chunk
            seen = tokens // c * (c * (c + 1) / 2) + (tokens % c) * (tokens % c + 1) / 2
            flops += 2.0 * seen * left.n_heads * (left.head_dim + left.v_dim)
            flops += 6.0 * tokens * right.n_heads * right.head_dim * right.v_dim
        return flops
