"""The Vulosun decoder: its typed configuration and its model assembled from parts.

config.json gives every size and every constant that differs between models of the design:

    architecture "Vulosun", vocab, width, norm.eps,
    layers: [{type: "parallel", mixer: {left: {heads, kv_heads, dim, vdim, scale, rot: {base, dims}},
                                        right: {heads, dim, vdim, decay: [..]}, left_scale, right_scale}, mlp: ...},
             {type: "attention", mixer: {heads, kv_heads, dim, vdim, scale, rot: {base, dims}}, mlp: ...},
             {type: "attention_2", mixer: {heads, kv_heads, dim, vdim, scale, diff, mask: {size},
                                           rot: {base, dims, scaling: {factor}}, kv_from: j or absent}, mlp: ...}, ...]
    mlp: null, {kind: "dense", ff} or
         {kind: "moe", router: {experts, top, scale, groups: {count, keep}}, expert: {ff}, shared: {ff} or absent}

A layer (`parts.SandwichBlock`) has a layer norm before and after each sublayer: x <- x + norm1b(mixer(norm1(x))); x <- x +
norm2b(ff(norm2(x))). Mixers, all built on `parts.ParallelMixer`: two mixers side by side, attention with queries and keys
normed per head, halves rotated and a sink per head (`parts.RotaryAttention`), and lightning attention
(`parts.LightningAttention`), added with a weight each; attention with whole-row norms, neighbours rotated and a gate per head
(`parts.RotaryAttention`); differential attention inside chunks of positions, with biases and gates
(`parts.DifferentialAttention`). A differential layer with `kv_from: j` reads layer j's keys and values: its schedule entry
names that layer's cache slot and writes nothing there. Feed-forwards: SiLU-gated (`parts.GatedFeedForward`), or routed experts
behind the square of relu, chosen among the best groups by sigmoid scores that also weigh their results, beside a shared expert
of the same form (`parts.RoutedExperts`, `parts.ReluSquaredFeedForward`), or none. Tensor names are the checkpoint's own:
`embed`, `l<i>.norm1`, `l<i>.norm1b.b`, `l<i>.mix.left.q.norm`, `l<i>.mix.left.sink`, `l<i>.mix.right.g`, `l<i>.mix.q.b`,
`l<i>.mix.lq1`, `l<i>.mlp.e<j>.up`, `l<i>.mlp.shared.down`, `final.norm.b`, `head`.
"""
from __future__ import annotations

from dataclasses import dataclass
import json

import torch

from ..config.model_config import ConfigError, eos_tuple
from ..config.registry import register_architecture
from ..parts import (DecoderModel, DifferentialAttention, GatedFeedForward, LayerNorm, LayerRun, LightningAttention, OutputHead,
                     ParallelMixer, ReluSquaredFeedForward, RotaryAttention, RotaryEmbedding, RoutedExperts, SandwichBlock,
                     TokenEmbedding)
from ..kernels.ops import MOE_MAX_EXPERTS

MIXERS = ("parallel", "attention", "attention_2")
NO_POSITION_LIMIT = 1 << 30      # the design has no learned positions: nothing bounds a request's length but the cache
MAX_HEAD = 256                   # key elements (of a differential head's two maps together) and value elements the kernels take


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


def _check_attention(m, where, i, maps=1):
    for key in ("heads", "kv_heads", "dim", "vdim"):
        _positive(_need(m, key, where), f"layer {i}: {key}")
    if m["heads"] % m["kv_heads"]:
        raise ConfigError(f"layer {i}: heads must be a multiple of kv_heads")
    if max(maps * m["dim"], m["vdim"]) > MAX_HEAD:
        raise ConfigError(f"layer {i}: the attention kernels take keys (all maps of a head together) and values of up to {MAX_HEAD} elements")
    _positive_float(_need(m, "scale", where), f"layer {i}: scale")
    rot = _need(m, "rot", where)
    dims = _positive(_need(rot, "dims", where + "rot."), f"layer {i}: rot.dims")
    if dims % 2 or dims > m["dim"]:
        raise ConfigError(f"layer {i}: rot.dims must be even and at most dim")
    _positive_float(_need(rot, "base", where + "rot."), f"layer {i}: rot.base")
    if rot.get("scaling") is not None:
        _positive_float(_need(rot["scaling"], "factor", where + "rot.scaling."), f"layer {i}: rot.scaling.factor")


def _same_cache(a, b):
    """Do two differential mixers agree in what lies in the pages?"""
    return all(a[k] == b[k] for k in ("heads", "kv_heads", "dim", "vdim", "rot"))


def _check_mixer(kind, layers, i):
    m, where = layers[i]["mixer"], f"layers[{i}].mixer."
    if kind == "parallel":
        left, right = _need(m, "left", where), _need(m, "right", where)
        _check_attention(left, where + "left.", i)
        for key in ("heads", "dim", "vdim"):
            _positive(_need(right, key, where + "right."), f"layer {i}: right.{key}")
        if right["dim"] > MAX_HEAD:
            raise ConfigError(f"layer {i}: the recurrence's kernels take keys of up to {MAX_HEAD} elements")
        decay = _need(right, "decay", where + "right.")
        if not isinstance(decay, list) or len(decay) != right["heads"]:
            raise ConfigError(f"layer {i}: right.decay must hold one number per head")
        for d in decay:
            if not 0 < _number(d, f"layer {i}: right.decay") <= 1:
                raise ConfigError(f"layer {i}: decays must lie in (0, 1], found {d!r}")
        for key in ("left_scale", "right_scale"):
            _number(_need(m, key, where), f"layer {i}: {key}")
        return
    _check_attention(m, where, i, maps=2 if kind == "attention_2" else 1)
    if kind == "attention":
        return
    _number(_need(m, "diff", where), f"layer {i}: diff")
    _positive(_need(_need(m, "mask", where), "size", where + "mask."), f"layer {i}: mask.size")
    source = m.get("kv_from")
    if source is None:
        return
    if isinstance(source, bool) or not isinstance(source, int) or not 0 <= source < i:
        raise ConfigError(f"layer {i}: kv_from must name an earlier layer, found {source!r}")
    other = layers[source]
    if other["type"] != kind or other["mixer"].get("kv_from") is not None:
        raise ConfigError(f"layer {i}: kv_from names layer {source}, which has no keys and values of its own of this kind")
    if not _same_cache(m, other["mixer"]):
        raise ConfigError(f"layer {i}: heads, sizes and rotation must equal those of layer {source}, whose keys and values it reads")


def _check_mlp(mlp, i):
    where = f"layers[{i}].mlp."
    kind = _need(mlp, "kind", where)
    if kind == "dense":
        _positive(_need(mlp, "ff", where), f"layer {i}: ff")
        return
    if kind != "moe":
        raise ConfigError(f"layer {i}: feed-forward kind {kind!r} is not built (known: 'dense', 'moe')")
    router, expert = _need(mlp, "router", where), _need(mlp, "expert", where)
    experts = _positive(_need(router, "experts", where + "router."), f"layer {i}: experts")
    top = _positive(_need(router, "top", where + "router."), f"layer {i}: top")
    _number(_need(router, "scale", where + "router."), f"layer {i}: router.scale")
    count, keep = _groups(router)
    _positive(count, f"layer {i}: groups.count")
    _positive(keep, f"layer {i}: groups.keep")
    if experts > MOE_MAX_EXPERTS or experts % count or keep > count or top > keep * (experts // count):
        raise ConfigError(f"layer {i}: at most {MOE_MAX_EXPERTS} experts in equal groups, of which those kept must hold `top`")
    _positive(_need(expert, "ff", where + "expert."), f"layer {i}: expert.ff")
    if mlp.get("shared") is not None:
        _positive(_need(mlp["shared"], "ff", where + "shared."), f"layer {i}: shared.ff")


def _groups(router):
    g = router.get("groups")
    return (_need(g, "count", "groups."), _need(g, "keep", "groups.")) if g is not None else (1, 1)


@dataclass(frozen=True)
class VulosunConfig:
    architecture: str
    vocab_size: int
    hidden_size: int
    norm_eps: float
    layers: tuple                 # the layer entries of config.json, as immutable JSON text each
    max_position_embeddings: int = NO_POSITION_LIMIT
    eos_token_ids: tuple = ()

    ARCHITECTURE = "Vulosun"
    MODEL_TYPE = "vulosun"

    @classmethod
    def from_dict(cls, d):
        if d.get("architecture", d.get("model_type")) not in (cls.ARCHITECTURE, cls.MODEL_TYPE):
            raise ConfigError(f"architecture {d.get('architecture')!r} is not {cls.ARCHITECTURE!r}")
        layers = _need(d, "layers", "")
        if not isinstance(layers, list) or not layers:
            raise ConfigError("'layers' must be a non-empty list")
        for i, layer in enumerate(layers):
            kind = _need(layer, "type", f"layers[{i}].")
            if kind not in MIXERS:
                raise ConfigError(f"layer {i}: mixer type {kind!r} is not built (known: {', '.join(MIXERS)})")
            _need(layer, "mixer", f"layers[{i}].")
            _check_mixer(kind, layers, i)
            if layer.get("mlp") is not None:
                _check_mlp(layer["mlp"], i)
        eps = _positive_float(_need(_need(d, "norm", ""), "eps", "norm."), "norm.eps")
        return cls(architecture=cls.ARCHITECTURE, vocab_size=_positive(_need(d, "vocab", ""), "vocab"),
                   hidden_size=_positive(_need(d, "width", ""), "width"), norm_eps=eps,
                   layers=tuple(json.dumps(layer, sort_keys=True) for layer in layers), eos_token_ids=eos_tuple(d.get("eos_token_id")))

    def layer_dicts(self):
        return [json.loads(text) for text in self.layers]

    def to_dict(self):
        d = {"architecture": self.architecture, "vocab": self.vocab_size, "width": self.hidden_size,
             "norm": {"eps": self.norm_eps}, "layers": self.layer_dicts()}
        if self.eos_token_ids:
            d["eos_token_id"] = list(self.eos_token_ids)
        return d

    def describe(self):
        return self.to_dict()


def _feed_forward(prefix, C, mlp):
    if mlp["kind"] == "dense":
        return GatedFeedForward([prefix + n for n in ("gate", "up", "down")], C, mlp["ff"], activation="silu", suffix="")
    router, shared = mlp["router"], mlp.get("shared")
    if shared is not None:
        shared = ReluSquaredFeedForward([prefix + "shared.up", prefix + "shared.down"], C, shared["ff"], suffix="")
    return RoutedExperts(prefix, C, router["experts"], router["top"], mlp["expert"]["ff"], shared=shared, kind="relu_squared",
                         weighting="sigmoid", groups=_groups(router), weight_scale=router["scale"])


def build_vulosun(config: VulosunConfig, packed=True):
    c = config
    C, eps, layers = c.hidden_size, c.norm_eps, c.layer_dicts()
    encodings = {}

    def rotary(rot, pairing):
        """One part per distinct encoding: its tables are formed once a step for all layers that share it."""
        factor = rot["scaling"]["factor"] if rot.get("scaling") is not None else 1.0
        key = (float(rot["base"]), int(rot["dims"]), float(factor), pairing)
        if key not in encodings:
            encodings[key] = RotaryEmbedding(rot["dims"], rot["base"], rot["dims"], pairing=pairing, divide=factor)
        return encodings[key]

    def norm(name):
        return LayerNorm(name, C, eps, suffixes=("", ".b"))

    # whose keys and values a layer reads, and the chunk sizes of everybody who reads a layer's
    source = [m["kv_from"] if m.get("kv_from") is not None else i for i, m in enumerate(lay["mixer"] for lay in layers)]
    blocks = []
    for i, layer in enumerate(layers):
        p, m, mlp = f"l{i}.", layer["mixer"], layer.get("mlp")
        if layer["type"] == "parallel":
            a, b = m["left"], m["right"]
            branches = [RotaryAttention(p + "mix.left.", a["heads"], a["kv_heads"], a["dim"], a["vdim"], rotary(a["rot"], "half"),
                                        a["scale"], eps, norm="head", sink=True),
                        LightningAttention(p + "mix.right.", b["heads"], b["dim"], b["vdim"], b["decay"], eps)]
            scales = [m["left_scale"], m["right_scale"]]
        elif layer["type"] == "attention":
            branches = [RotaryAttention(p + "mix.", m["heads"], m["kv_heads"], m["dim"], m["vdim"], rotary(m["rot"], "adjacent"),
                                        m["scale"], eps, norm="row", gate=True)]
            scales = [1.0]
        else:
            retain = [layers[j]["mixer"]["mask"]["size"] for j in range(len(layers))
                      if layers[j]["type"] == "attention_2" and source[j] == source[i]]
            branches = [DifferentialAttention(p + "mix.", m["heads"], m["kv_heads"], m["dim"], m["vdim"], rotary(m["rot"], "adjacent"),
                                              m["scale"], eps, m["diff"], chunk=m["mask"]["size"], retain=retain,
                                              reads_other=source[i] != i)]
            scales = [1.0]
        mixer = ParallelMixer(C, branches, scales, proj_dtype=torch.float32)
        ffn = _feed_forward(p + "mlp.", C, mlp) if mlp is not None else None
        unused = [p + n for n in ("norm2", "norm2.b", "norm2b", "norm2b.b")] if ffn is None else []
        blocks.append(SandwichBlock(C, mixer, (norm(p + "norm1"), norm(p + "norm1b")), ffn,
                                    (norm(p + "norm2"), norm(p + "norm2b")) if ffn is not None else None, unused_names=unused))
    for before, after in zip(blocks, blocks[1:]):
        before.next_norm = after.mixer_norm
    # a layer that reads another's keys and values runs on that layer's cache slot; every other layer has a slot of its own
    slots = {i: k for k, i in enumerate(j for j in range(len(layers)) if source[j] == j)}
    schedule = [LayerRun(i, slots[source[i]], writes_cache=source[i] == i) for i in range(len(layers))]
    embedding = TokenEmbedding("embed", c.vocab_size, C, suffix="")
    head = OutputHead("head", c.vocab_size, C, suffix="")
    return DecoderModel(c, embedding, blocks, norm("final.norm"), head, schedule=schedule)


register_architecture(VulosunConfig.ARCHITECTURE, VulosunConfig.MODEL_TYPE, VulosunConfig, build_vulosun, replace=True)
