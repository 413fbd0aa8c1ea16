"""The Darolix decoder: its typed configuration and its model assembled from parts.

config.json gives every size and every constant that differs between models of the design:

    architecture "Darolix", vocab, width, norm.eps, embedding.scale, loop: {start, stop, times} (optional),
    layers: [{type: "mamba2", mixer: {heads, vdim, state, groups, conv, norm_groups}, mlp: ...},
             {type: "parallel", mixer: {left: {heads, kv_heads, dim, vdim, scale, softcap, q_temp: {coef, every}},
                                        right: {heads, dim, vdim, tau}}, mlp: ...}, ...]
    mlp: null or {kind: "moe", router: {experts, identity, top}, expert: {ff}}

The rank of the linear attention's decay is the one size config.json leaves to the checkpoint: it is the number of rows of
`l<i>.mix.right.a1` (`with_tensor_shapes`); where there is no checkpoint yet (random weights), `right.rank` or DECAY_RANK.

A layer (`parts.ParallelBlock`, shared norm) has one RMS norm whose result both sublayers read: x <- x + (mixer(h) + ff(h)),
h = norm1(x). Mixers: the Mamba-2 state-space recurrence behind a short convolution (`parts.StateSpace`); or two mixers side
by side (`parts.ParallelMixer` with a norm on each result, half of each): attention without a rotation, with normed heads,
a query temperature that grows with the position and a soft cap (`parts.NormedAttention`), and gated linear attention
(`parts.GatedLinearAttention`). Feed-forward: routed SiLU-gated experts scored by a softmax over all of them, chosen with a
correction, the last ones identities (`parts.RoutedExperts`), or none. Embedding: scaled rows plus fixed sinusoids
(`parts.SinusoidalEmbedding`). `loop` runs layers start .. stop - 1 `times` times in a row with the same weights; every
pass has a cache slot (pages, state) of its own, and before each pass but the first the embedding's output is added to the
stream (`LayerRun.adds_embedding`). Tensor names are the checkpoint's own: `embed`, `l<i>.norm1`, `l<i>.mix.in`,
`l<i>.mix.conv.b`, `l<i>.mix.left.q`, `l<i>.mix.right.a2.b`, `l<i>.mix.left.out`, `l<i>.mlp.e<j>.gate`,
`l<i>.mlp.correction`, `final.norm`, `head`.

Constants the design fixes (not in config.json) live in the parts or below: the sinusoids' 10000, the half of each mixer's
result, the linear attention's dim^-1/2 and the router's 1e-20.
"""
from __future__ import annotations

from dataclasses import dataclass, replace
import json

import torch

from ..config.model_config import ConfigError, eos_tuple
from ..config.registry import register_architecture
from ..parts import (DecoderModel, GatedLinearAttention, LayerRun, NormedAttention, OutputHead, ParallelBlock, ParallelMixer,
                     RMSNorm, RoutedExperts, SinusoidalEmbedding, StateSpace)
from ..kernels.ops import CONV_MAX_TAPS, MOE_MAX_EXPERTS

MIXERS = ("mamba2", "parallel")
NO_POSITION_LIMIT = 1 << 30      # nothing bounds a request's length but the cache
DECAY_RANK = 16                  # of models drawn at random whose configuration does not say
BRANCH_WEIGHT = 0.5              # of each of the two mixers' normed results


def _need(d, key, where):
    if not isinstance(d, dict) or key not in d:
        raise ConfigError(f"config.json lacks {where}{key!r}")
    return d[key]


def _positive(value, what):
    if isinstance(value, bool) or not isinstance(value, int) or value <= 0:
        raise ConfigError(f"{what} must be a positive integer, found {value!r}")
    return value


def _number(value, what):
    if isinstance(value, bool) or not isinstance(value, (int, float)):
        raise ConfigError(f"{what} must be a number, found {value!r}")
    return float(value)


def _positive_float(value, what):
    if not _number(value, what) > 0:
        raise ConfigError(f"{what} must be positive, found {value!r}")
    return float(value)


def _check_mixer(kind, m, i):
    where = f"layers[{i}].mixer."
    if kind == "mamba2":
        for key in ("heads", "vdim", "state", "groups", "norm_groups", "conv"):
            _positive(_need(m, key, where), f"layer {i}: {key}")
        if m["heads"] % m["groups"]:
            raise ConfigError(f"layer {i}: heads must be a multiple of groups")
        if (m["heads"] * m["vdim"]) % m["norm_groups"]:
            raise ConfigError(f"layer {i}: norm_groups must divide heads * vdim")
        if m["state"] > 256:
            raise ConfigError(f"layer {i}: the recurrence's kernels take states of up to 256 elements")
        if m["conv"] > CONV_MAX_TAPS:
            raise ConfigError(f"layer {i}: a convolution has at most {CONV_MAX_TAPS} taps")
        return
    left, right = _need(m, "left", where), _need(m, "right", where)
    for key in ("heads", "kv_heads", "dim", "vdim"):
        _positive(_need(left, key, where + "left."), f"layer {i}: left.{key}")
    if left["heads"] % left["kv_heads"]:
        raise ConfigError(f"layer {i}: left.heads must be a multiple of left.kv_heads")
    if max(left["dim"], left["vdim"]) > 256:
        raise ConfigError(f"layer {i}: the attention kernels take key and value sizes up to 256")
    _positive_float(_need(left, "scale", where + "left."), f"layer {i}: left.scale")
    if left.get("softcap"):
        _positive_float(left["softcap"], f"layer {i}: left.softcap")
    if left.get("q_temp") is not None:
        _number(_need(left["q_temp"], "coef", where + "left.q_temp."), f"layer {i}: left.q_temp.coef")
        _positive(_need(left["q_temp"], "every", where + "left.q_temp."), f"layer {i}: left.q_temp.every")
    for key in ("heads", "dim", "vdim"):
        _positive(_need(right, key, where + "right."), f"layer {i}: right.{key}")
    if right["dim"] > 256:
        raise ConfigError(f"layer {i}: the recurrence's kernels take keys of up to 256 elements")
    _positive_float(_need(right, "tau", where + "right."), f"layer {i}: right.tau")
    if right.get("rank") is not None:
        _positive(right["rank"], f"layer {i}: right.rank")


def _check_mlp(mlp, i):
    where = f"layers[{i}].mlp."
    if _need(mlp, "kind", where) != "moe":
        raise ConfigError(f"layer {i}: feed-forward kind {mlp['kind']!r} is not built (known: 'moe')")
    router, expert = _need(mlp, "router", where), _need(mlp, "expert", where)
    experts = _positive(_need(router, "experts", where + "router."), f"layer {i}: experts")
    top = _positive(_need(router, "top", where + "router."), f"layer {i}: top")
    identity = router.get("identity") or 0
    if isinstance(identity, bool) or not isinstance(identity, int) or identity < 0:
        raise ConfigError(f"layer {i}: identity must be an integer, zero or more")
    if top > experts + identity or experts + identity > MOE_MAX_EXPERTS:
        raise ConfigError(f"layer {i}: top must not exceed the experts, and these not {MOE_MAX_EXPERTS}")
    _positive(_need(expert, "ff", where + "expert."), f"layer {i}: expert.ff")


@dataclass(frozen=True)
class DarolixConfig:
    architecture: str
    vocab_size: int
    hidden_size: int
    norm_eps: float
    embedding_scale: float
    loop: tuple                   # (start, stop, times); (0, 0, 1) when nothing repeats
    layers: tuple                 # the layer entries of config.json, as immutable JSON text each
    decay_ranks: tuple            # per layer, of the linear attention's decay (0 where a layer has none)
    max_position_embeddings: int = NO_POSITION_LIMIT
    eos_token_ids: tuple = ()

    ARCHITECTURE = "Darolix"
    MODEL_TYPE = "darolix"

    @classmethod
    def from_dict(cls, d):
        if d.get("architecture", d.get("model_type")) not in (cls.ARCHITECTURE, cls.MODEL_TYPE):
            raise ConfigError(f"architecture {d.get('architecture')!r} is not {cls.ARCHITECTURE!r}")
        layers = _need(d, "layers", "")
        if not isinstance(layers, list) or not layers:
            raise ConfigError("'layers' must be a non-empty list")
        ranks = []
        for i, layer in enumerate(layers):
            kind = _need(layer, "type", f"layers[{i}].")
            if kind not in MIXERS:
                raise ConfigError(f"layer {i}: mixer type {kind!r} is not built (known: {', '.join(MIXERS)})")
            mixer = _need(layer, "mixer", f"layers[{i}].")
            _check_mixer(kind, mixer, i)
            if layer.get("mlp") is not None:
                _check_mlp(layer["mlp"], i)
            ranks.append((mixer["right"].get("rank") or DECAY_RANK) if kind == "parallel" else 0)
        loop = d.get("loop")
        start, stop, times = 0, 0, 1
        if loop is not None:
            start, stop, times = (_need(loop, key, "loop.") for key in ("start", "stop", "times"))
            for v in (start, stop, times):
                if isinstance(v, bool) or not isinstance(v, int):
                    raise ConfigError("loop.start, loop.stop and loop.times must be integers")
            if not (0 <= start <= stop <= len(layers)) or times < 1:
                raise ConfigError("loop must name layers start .. stop - 1 of the model and run them at least once")
        eps = _positive_float(_need(_need(d, "norm", ""), "eps", "norm."), "norm.eps")
        scale = _number(_need(_need(d, "embedding", ""), "scale", "embedding."), "embedding.scale")
        return cls(architecture=cls.ARCHITECTURE, vocab_size=_positive(_need(d, "vocab", ""), "vocab"),
                   hidden_size=_positive(_need(d, "width", ""), "width"), norm_eps=eps, embedding_scale=scale,
                   loop=(start, stop, times), layers=tuple(json.dumps(layer, sort_keys=True) for layer in layers),
                   decay_ranks=tuple(ranks), eos_token_ids=eos_tuple(d.get("eos_token_id")))

    def with_tensor_shapes(self, shapes):
        """The same with every decay's rank as the checkpoint's tensors have it (absent ones are the loader's to report)."""
        ranks = []
        for i, rank in enumerate(self.decay_ranks):
            shape = shapes.get(f"l{i}.mix.right.a1")
            ranks.append(int(shape[0]) if rank and shape is not None and len(shape) == 2 else rank)
        return replace(self, decay_ranks=tuple(ranks))

    def layer_dicts(self):
        return [json.loads(text) for text in self.layers]

    def layer_runs(self):
        """[(layer, does a pass but the first begin here)] in the order the layers run."""
        start, stop, times = self.loop
        runs = [(i, False) for i in range(start)]
        for turn in range(times):
            runs += [(i, turn > 0 and i == start) for i in range(start, stop)]
        return runs + [(i, False) for i in range(stop, len(self.layers))]

    def to_dict(self):
        d = {"architecture": self.architecture, "vocab": self.vocab_size, "width": self.hidden_size,
             "norm": {"eps": self.norm_eps}, "embedding": {"scale": self.embedding_scale}, "layers": self.layer_dicts()}
        if self.loop != (0, 0, 1):
            d["loop"] = dict(zip(("start", "stop", "times"), self.loop))
        if self.eos_token_ids:
            d["eos_token_id"] = list(self.eos_token_ids)
        return d

    def describe(self):
        return self.to_dict()


def build_darolix(config: DarolixConfig, packed=True):
    c = config
    C = c.hidden_size

    def norm(name):
        return RMSNorm(name, C, c.norm_eps, suffix="")

    blocks = []
    for i, layer in enumerate(c.layer_dicts()):
        p, m, mlp = f"l{i}.", layer["mixer"], layer.get("mlp")
        if layer["type"] == "mamba2":
            mixer = StateSpace(p + "mix.", C, m["heads"], m["vdim"], m["state"], m["groups"], m["conv"], m["norm_groups"],
                               c.norm_eps)
        else:
            a, b = m["left"], m["right"]
            temperature = (a["q_temp"]["coef"], a["q_temp"]["every"]) if a.get("q_temp") is not None else None
            left = NormedAttention(p + "mix.left.", a["heads"], a["kv_heads"], a["dim"], a["vdim"], a["scale"], c.norm_eps,
                                   softcap=a.get("softcap") or None, temperature=temperature)
            right = GatedLinearAttention(p + "mix.right.", b["heads"], b["dim"], b["vdim"], c.decay_ranks[i], b["tau"], c.norm_eps)
            mixer = ParallelMixer(C, [left, right], [BRANCH_WEIGHT, BRANCH_WEIGHT], proj_dtype=torch.float32,
                                  result_norms=[norm(p + "mix.left.out"), norm(p + "mix.right.out")])
        ffn = None
        if mlp is not None:
            router = mlp["router"]
            ffn = RoutedExperts(p + "mlp.", C, router["experts"], router["top"], mlp["expert"]["ff"], kind="silu",
                                weighting="softmax_all", correction="correction", identity=router.get("identity") or 0)
        blocks.append(ParallelBlock(C, norm(p + "norm1"), mixer, ffn=ffn, shared_norm=True))
    # every run of a layer has a cache slot of its own: a repeated layer shares its weights, not its pages or state
    runs = c.layer_runs()
    schedule = [LayerRun(block, slot, adds_embedding=again) for slot, (block, again) in enumerate(runs)]
    embedding = SinusoidalEmbedding("embed", c.vocab_size, C, scale=c.embedding_scale, suffix="",
                                    keep=any(again for _, again in runs))
    head = OutputHead("head", c.vocab_size, C, suffix="")
    return DecoderModel(c, embedding, blocks, norm("final.norm"), head, schedule=schedule)


register_architecture(DarolixConfig.ARCHITECTURE, DarolixConfig.MODEL_TYPE, DarolixConfig, build_darolix, replace=True)
