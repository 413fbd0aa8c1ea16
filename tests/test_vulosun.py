"""The Vulosun design without a GPU: configuration, registry, tensor names, cache needs (chunked groups, layers that read
another's pages) and schedule, the command line, and the plain implementation's mechanisms against closed forms (so that the
oracle the GPU tests use is itself pinned)."""
import json
import math

import numpy as np
import pytest
import torch

import plain_vulosun as plain
from vulosun_util import CONFIGS, make_weights, tensor_shapes, write_folder


@pytest.mark.parametrize("name", list(CONFIGS))
def test_config_registry_and_tensor_names(name, tmp_path):
    from tessweave_engine_amd.config import build_model, config_from_dict, read_model_config
    c = CONFIGS[name]
    config_ = config_from_dict(c)
    assert config_.architecture == "Vulosun" and config_.vocab_size == c["vocab"]
    assert config_from_dict(config_.to_dict()) == config_
    folder = write_folder(tmp_path, c, make_weights(c, 0))
    assert read_model_config(folder) == config_
    specs = {s.name: s.shape for s in build_model(config_).tensor_specs() if s.optional_alias_of is None}
    assert specs == tensor_shapes(c)


def test_weights_load_with_and_without_unused_norms(tmp_path):
    """A layer without a feed-forward may come with the norms it would have had; anything else is reported."""
    from tessweave_engine_amd.weights import WeightError, load_model
    c = CONFIGS["one"]
    weights = make_weights(c, 0)
    load_model(write_folder(tmp_path / "a", c, weights), dtype="float32", device="cpu")
    for name in ("norm2", "norm2.b", "norm2b", "norm2b.b"):
        weights["l0." + name] = torch.zeros(50, dtype=torch.bfloat16)
    load_model(write_folder(tmp_path / "b", c, weights), dtype="float32", device="cpu")
    del weights["l0.mix.left.sink"]
    weights["l0.mix.left.g"] = torch.zeros(2, 50, dtype=torch.bfloat16)
    with pytest.raises(WeightError, match="(?s)missing .*l0.mix.left.sink.*unexpected .*l0.mix.left.g"):
        load_model(write_folder(tmp_path / "c", c, weights), dtype="float32", device="cpu")


def test_config_rejections():
    from tessweave_engine_amd.config import ConfigError, config_from_dict
    base = json.loads(json.dumps(CONFIGS["odd"]))
    for change in (lambda c: c["layers"][0].__setitem__("type", "other"),
                   lambda c: c["layers"][0]["mixer"].pop("diff"),
                   lambda c: c["layers"][0]["mixer"].pop("mask"),
                   lambda c: c["layers"][0]["mixer"]["mask"].__setitem__("size", 0),
                   lambda c: c["layers"][0]["mixer"].__setitem__("dim", 129),
                   lambda c: c["layers"][0]["mixer"].__setitem__("kv_from", 0),
                   lambda c: c["layers"][2]["mixer"].__setitem__("kv_from", 1),
                   lambda c: c["layers"][3]["mixer"].__setitem__("kv_from", 2),
                   lambda c: c["layers"][2]["mixer"].__setitem__("kv_from", True),
                   lambda c: c["layers"][2]["mixer"]["rot"].__setitem__("base", 3.0),
                   lambda c: c["layers"][2]["mixer"].__setitem__("vdim", 24),
                   lambda c: c["layers"][1]["mixer"].__setitem__("kv_heads", 4),
                   lambda c: c["layers"][1]["mixer"].__setitem__("scale", 0),
                   lambda c: c["layers"][1]["mixer"]["rot"].__setitem__("dims", 26),
                   lambda c: c["layers"][1]["mixer"]["rot"].__setitem__("dims", 5),
                   lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].__setitem__("factor", -1.0),
                   lambda c: c["layers"][4]["mixer"].pop("left_scale"),
                   lambda c: c["layers"][4]["mixer"]["right"]["decay"].pop(),
                   lambda c: c["layers"][4]["mixer"]["right"]["decay"].__setitem__(0, 1.5),
                   lambda c: c["layers"][4]["mixer"]["right"]["decay"].__setitem__(0, 0),
                   lambda c: c["layers"][4]["mixer"]["right"].__setitem__("dim", 257),
                   lambda c: c["layers"][1]["mlp"].__setitem__("kind", "other"),
                   lambda c: c["layers"][0]["mlp"]["router"].__setitem__("top", 5),
                   lambda c: c["layers"][0]["mlp"]["router"]["groups"].__setitem__("count", 4),
                   lambda c: c["layers"][0]["mlp"]["router"]["groups"].__setitem__("keep", 7),
                   lambda c: c["layers"][0]["mlp"]["router"].pop("scale"),
                   lambda c: c["layers"][0]["mlp"]["shared"].__setitem__("ff", 0),
                   lambda c: c["norm"].__setitem__("eps", 0)):
        c = json.loads(json.dumps(base))
        change(c)
        with pytest.raises(ConfigError):
            config_from_dict(c)


def test_cache_layout_and_schedule():
    """A layer that reads another's keys and values runs on that layer's cache slot and writes nothing there; the slot is
    held for the chunks of all its readers; parallel layers page keys and values and hold the linear attention's state."""
    from tessweave_engine_amd.config import build_model, config_from_dict
    model = build_model(config_from_dict(CONFIGS["odd"]))
    assert [(r.block, r.cache_slot, r.writes_cache) for r in model.schedule] == \
        [(0, 0, True), (1, 1, True), (2, 0, False), (3, 0, False), (4, 2, True)]
    assert model.graph_safe_model and model.defers_sums
    layout = model.cache_layout()
    a, b, c = (need.paged for need in layout.needs)
    assert (a.kv_heads, a.head_dim, a.chunks, a.keeps_all) == (3, 32, (6, 10, 17), False)
    assert (b.kv_heads, b.head_dim, b.chunks, b.keeps_all) == (2, 48, (), True)
    assert (c.kv_heads, c.head_dim) == (3, 32) and dict(layout.needs[2].states)["lightning_attention.s"].shape == (3, 32, 32)
    assert not layout.shares_prefixes
    for before, after in zip(model.blocks, model.blocks[1:]):
        assert before.next_norm is after.mixer_norm
    wide = build_model(config_from_dict(CONFIGS["wide"]))
    assert [n.paged.chunks for n in wide.cache_layout().needs] == [(), (1000,), (32,), ()]
    # layers with the same encoding share a part (its tables are formed once a step), others do not
    encodings = [b.mixer.branches[0].position for b in model.blocks]
    assert encodings[0] is encodings[2] is encodings[3] and len({id(e) for e in encodings}) == 3


@pytest.mark.parametrize("chunks", [(1,), (7,), (16,), (24,), (6, 10, 17), (10, 15)])
def test_pages_of_chunks_come_back(chunks):
    """At every length, exactly the pages that some later query of some reader may see are held; promises are never exceeded."""
    from tessweave_engine_amd.cache import CacheManager
    from tessweave_engine_amd.cache.spec import CacheLayout, CacheNeed, PagedKV
    spec = PagedKV(2, 16, chunks=chunks)
    positions = np.arange(200)
    first = np.minimum.reduce([positions // c * c for c in chunks])
    assert (spec.first_position(positions) == first).all() and spec.first_position(37) == first[37]
    layout = CacheLayout([CacheNeed(paged=spec), CacheNeed(paged=PagedKV(2, 16))])
    page = 4
    m = CacheManager(layout, page, [60, 60], 2, prefix_cache=True)
    assert not m.prefix_cache
    seq = m.open("a")
    m.reserve(seq, 160, 5)
    at = 0
    for n in [1] * 30 + [5, 3, 2] * 13:
        m.ensure(seq, at + n)
        held = {b for b, p in enumerate(seq.tables[0]) if p >= 0}
        assert held >= set(range(first[at] // page, (at + n - 1) // page + 1))
        at += n
        m.advance(seq, at)
        m.check()
        held = {b for b, p in enumerate(seq.tables[0]) if p >= 0}
        assert held == set(range(first[at] // page, (at + page - 1) // page)) and seq.held(1) == (at + page - 1) // page
    m.close(seq)
    m.check()
    assert len(m.pools[0].free) == 60


def test_chunks_take_the_place_of_a_window():
    from tessweave_engine_amd.cache.spec import PagedKV
    for wrong in (dict(window=5, chunks=(4,)), dict(chunks=(0,))):
        with pytest.raises(ValueError):
            PagedKV(1, 16, **wrong)
    assert PagedKV(1, 16, chunks=[9, 4, 9]).chunks == (4, 9)
    window = PagedKV(1, 16, window=10)
    assert [window.first_position(p) for p in (0, 9, 10, 30)] == [0, 0, 1, 21] and window.span == 10


def test_random_weights_and_inspect_on_the_command_line(tmp_path, capsys):
    from tessweave_engine_amd.cli import main
    from tessweave_engine_amd.config import read_model_config
    source = tmp_path / "config.json"
    source.write_text(json.dumps(CONFIGS["odd"]))
    folder = tmp_path / "model"
    assert main(["random-weights", str(source), str(folder), "--seed", "3"]) == 0
    assert read_model_config(folder).to_dict()["layers"] == CONFIGS["odd"]["layers"]
    from safetensors import safe_open
    with safe_open(str(folder / "model.safetensors"), framework="pt") as f:
        assert {k: tuple(f.get_slice(k).get_shape()) for k in f.keys()} == tensor_shapes(CONFIGS["odd"])
    capsys.readouterr()
    assert main(["inspect", str(folder), "--kv-blocks", "10", "--block-size", "16"]) == 0
    shown = json.loads(capsys.readouterr().out)
    assert shown["architecture"]["architecture"] == "Vulosun" and [6, 10, 17] in [g.get("chunks") for g in shown["cache_groups"]]


# ---- the plain implementation's mechanisms against closed forms --------------------------------------------

F64 = torch.float64


def test_layer_norm_and_rms_norm():
    x = torch.tensor([[1.0, 3.0, 5.0, 7.0]], dtype=F64)
    w, b = torch.tensor([1.0, 2.0, 1.0, 1.0], dtype=F64), torch.tensor([0.0, 0.0, 5.0, 0.0], dtype=F64)
    s = math.sqrt(5.0 + 0.25)
    assert torch.allclose(plain.layer_norm(x, w, b, 0.25), torch.tensor([[-3 / s, -2 / s, 5 + 1 / s, 3 / s]], dtype=F64))
    assert torch.allclose(plain.rms_norm(x, w, 4.0), x * w / 5.0)


def test_rotations():
    """Which elements turn together, by which angles, and that the rest pass unchanged."""
    x = torch.arange(1.0, 8.0, dtype=F64).view(1, 1, 7).expand(4, 1, 7)
    r = {"base": 100.0, "dims": 4}
    near, half = plain.rotate_neighbours(x, r), plain.rotate_halves(x, r)
    for p in range(4):
        for out, pairs in ((near, [(0, 1), (2, 3)]), (half, [(0, 2), (1, 3)])):
            for i, (u, v) in enumerate(pairs):
                a = p * 100.0 ** (-2 * i / 4)
                assert out[p, 0, u].item() == pytest.approx((u + 1) * math.cos(a) - (v + 1) * math.sin(a))
                assert out[p, 0, v].item() == pytest.approx((v + 1) * math.cos(a) + (u + 1) * math.sin(a))
            assert out[p, 0, 4:].tolist() == [5, 6, 7]
    scaled = plain.rotate_neighbours(x, dict(r, scaling={"factor": 3.0}))
    assert torch.allclose(scaled[3], near[1])


def test_masks_and_sinks():
    seen = plain.same_chunk(7, 3)
    assert [row.nonzero().flatten().tolist() for row in seen] == [[0], [0, 1], [0, 1, 2], [3], [3, 4], [3, 4, 5], [6]]
    T = 4
    q, v = torch.zeros(T, 2, 3, dtype=F64), torch.ones(T, 1, 1, dtype=F64)
    k = torch.randn(T, 1, 3, generator=torch.Generator().manual_seed(0), dtype=F64)
    sink = torch.tensor([0.0, math.log(3.0)], dtype=F64)
    o = plain.attend(q, k, v, 0.7, plain.causal(T), sink)        # t + 1 scores of zero and the sink
    for t in range(T):
        assert o[t, 0, 0].item() == pytest.approx((t + 1) / (t + 2)) and o[t, 1, 0].item() == pytest.approx((t + 1) / (t + 4))
    assert torch.allclose(plain.attend(q, k, v, 0.7, plain.causal(T)), torch.ones(T, 2, 1, dtype=F64))


def test_whole_row_norm_and_gates():
    """Norm over all heads at once (one head's size moves the other's), and one gate per head on its result."""
    C = 4
    g = torch.Generator().manual_seed(2)
    m = {"heads": 2, "kv_heads": 1, "dim": 2, "vdim": 2, "scale": 1.0, "rot": {"base": 10.0, "dims": 2}}
    eye = torch.eye(C, dtype=F64)
    w = {"q": eye, "k": torch.zeros(2, C, dtype=F64), "v": torch.randn(2, C, generator=g, dtype=F64), "q.norm": torch.ones(4, dtype=F64),
         "k.norm": torch.ones(2, dtype=F64), "g": torch.tensor([[1.0, 0, 0, 0], [0, 2.0, 0, 0]], dtype=F64), "o": eye}
    h = torch.randn(1, C, generator=g, dtype=F64)
    o = plain.whole_normed_attention(h, w, m, 1e-5).view(2, 2)
    v = (h @ w["v"].T)[0]
    assert torch.allclose(o[0], v * torch.sigmoid(h[0, 0])) and torch.allclose(o[1], v * torch.sigmoid(2 * h[0, 1]))


def test_differential_closed_forms():
    w = {"lq1": torch.tensor([1.0, 2.0], dtype=F64), "lk1": torch.tensor([0.5, 0.1], dtype=F64),
         "lq2": torch.tensor([1.0, 0.0], dtype=F64), "lk2": torch.tensor([-1.0, 5.0], dtype=F64)}
    lam = plain.differential_lambda(w, 0.3)
    assert lam.item() == pytest.approx(math.exp(0.7) - math.exp(-1.0) + 0.3)
    a1, a2 = torch.tensor([3.0, 1.0], dtype=F64), torch.tensor([1.0, 2.0], dtype=F64)
    o = plain.combine_maps(a1, a2, 2.0, 0.25, 0.0)
    assert torch.allclose(o, 0.75 * torch.tensor([1.0, -3.0], dtype=F64) / math.sqrt(5.0))


def test_shared_keys_and_values():
    """A layer that reads another's takes its keys (rotated) and values as they are, with its own queries and chunks."""
    g = torch.Generator().manual_seed(4)
    T, C = 6, 5
    m = {"heads": 2, "kv_heads": 1, "dim": 2, "vdim": 3, "scale": 0.5, "rot": {"base": 10.0, "dims": 2}, "mask": {"size": 2}, "diff": 0.2}
    w = {n: torch.randn(s, generator=g, dtype=F64) for n, s in
         {"q": (8, C), "q.b": (8,), "k": (4, C), "k.b": (4,), "v": (3, C), "v.b": (3,), "g": (2, C), "o": (C, 6),
          "lq1": (2,), "lk1": (2,), "lq2": (2,), "lk2": (2,)}.items()}
    h, other = torch.randn(T, C, generator=g, dtype=F64), torch.randn(T, C, generator=g, dtype=F64)
    kv = plain.chunked_keys_values(other, w, m)
    wide = dict(m, mask={"size": 3})
    got = plain.differential_attention(h, w, wide, 1e-5, kv)
    k, v = kv
    q = plain.rotate_neighbours((h @ w["q"].T + w["q.b"]).view(T, 4, 2), m["rot"])
    for t in range(T):
        lo = t // 3 * 3
        out = []
        for a in range(2):
            maps = []
            for i in range(2):
                s = torch.softmax((k[lo:t + 1, 0, i] @ q[t, 2 * a + i]) * 0.5, 0)
                maps.append(s @ v[lo:t + 1, 0])
            o = maps[0] - plain.differential_lambda(w, 0.2) * maps[1]
            out.append(o / torch.sqrt((o * o).mean() + 1e-5) * 0.8 * torch.sigmoid(h[t] @ w["g"][a]))
        assert torch.allclose(got[t], torch.cat(out) @ w["o"].T)


def test_lightning_closed_form():
    T, D, E = 6, 3, 2
    g = torch.Generator().manual_seed(5)
    q, k, v = (torch.randn(T, n, generator=g, dtype=F64) for n in (D, D, E))
    o = plain.lightning_steps(q, k, v, 0.7)
    for t in range(T):
        assert torch.allclose(o[t], sum(0.7 ** (t - j) * (q[t] @ k[j]) * v[j] for j in range(t + 1)))
    m = {"heads": 1, "dim": 1, "vdim": 1, "decay": [0.5]}
    one = torch.ones(1, 1, dtype=F64)
    w = {"q": one, "k": one, "v": one, "g": one, "norm": torch.tensor([2.0], dtype=F64), "o": one}
    h = torch.tensor([[1.0], [2.0]], dtype=F64)
    s1, s2 = 1 / (1 + math.exp(-1)), 2 / (1 + math.exp(-2))
    o2 = s2 * (0.5 * s1 * s1 + s2 * s2)
    want = 2 * o2 / math.sqrt(o2 * o2 + 1e-5) / (1 + math.exp(-2))
    assert plain.lightning_attention(h, w, m, 1e-5)[1, 0].item() == pytest.approx(want)


def test_groups_of_experts():
    """The group with the largest single score is left out when the sums of the two largest say so; weights are the scaled
    scores as they are; margins of both choices."""
    s = torch.tensor([[0.9, 0.1, 0.2, 0.6, 0.55, 0.1]], dtype=F64)         # sums 1.1 and 1.15
    ids, margin = plain.choose_experts(s, {"experts": 6, "top": 2, "groups": {"count": 2, "keep": 1}})
    assert ids.tolist() == [[3, 4]] and margin.item() == pytest.approx(0.05)
    ids, margin = plain.choose_experts(s, {"experts": 6, "top": 2, "groups": {"count": 2, "keep": 2}})
    assert ids.tolist() == [[0, 3]] and margin.item() == pytest.approx(0.05)
    ids, margin = plain.choose_experts(s, {"experts": 6, "top": 3, "groups": {"count": 6, "keep": 3}})
    assert sorted(ids[0].tolist()) == [0, 3, 4] and margin.item() == pytest.approx(0.35)
    g = torch.Generator().manual_seed(0)
    C = 3
    w = {"router": torch.randn(4, C, generator=g, dtype=F64), "shared.up": torch.randn(2, C, generator=g, dtype=F64),
         "shared.down": torch.randn(C, 2, generator=g, dtype=F64)}
    for e in range(4):
        w[f"e{e}.up"], w[f"e{e}.down"] = torch.randn(5, C, generator=g, dtype=F64), torch.randn(C, 5, generator=g, dtype=F64)
    h = torch.randn(1, C, generator=g, dtype=F64)
    mlp = {"router": {"experts": 4, "top": 2, "scale": 1.5}, "expert": {"ff": 5}, "shared": {"ff": 2}}
    s = torch.sigmoid(h @ w["router"].T)[0]
    want = torch.clamp(h @ w["shared.up"].T, min=0) ** 2 @ w["shared.down"].T
    for e in torch.topk(s, 2).indices.tolist():
        want = want + 1.5 * s[e] * (torch.clamp(h @ w[f"e{e}.up"].T, min=0) ** 2 @ w[f"e{e}.down"].T)
    assert torch.allclose(plain.routed_ff(h, w, mlp), want)


def test_layer_arrangement():
    """A norm before and after each sublayer, both with biases; the weights of the two mixers side by side; kv_from."""
    c = CONFIGS["odd"]
    weights = {k: v.double() for k, v in make_weights(c, 2).items()}
    toks = [3, 50, 7, 7, 90, 1, 200, 4, 9, 10, 11, 12]
    layers = []
    logits = plain.forward(c, weights, toks, layers_out=layers)
    eps = c["norm"]["eps"]

    def norm(x, name):
        return plain.layer_norm(x, weights[name], weights[name + ".b"], eps)
    x = layers[1]
    held = plain.chunked_keys_values(norm(weights["embed"][toks], "l0.norm1"), plain.sub(weights, "l0.mix."), c["layers"][0]["mixer"])
    y = plain.differential_attention(norm(x, "l2.norm1"), plain.sub(weights, "l2.mix."), c["layers"][2]["mixer"], eps, held)
    x = x + norm(y, "l2.norm1b")
    x = x + norm(plain.routed_ff(norm(x, "l2.norm2"), plain.sub(weights, "l2.mlp."), c["layers"][2]["mlp"]), "l2.norm2b")
    assert torch.allclose(layers[2], x)
    h = norm(layers[3], "l4.norm1")
    m = c["layers"][4]["mixer"]
    y = 1.3 * plain.head_normed_attention(h, plain.sub(weights, "l4.mix.left."), m["left"], eps) + \
        0.7 * plain.lightning_attention(h, plain.sub(weights, "l4.mix.right."), m["right"], eps)
    assert torch.allclose(layers[4], layers[3] + norm(y, "l4.norm1b"))
    assert torch.allclose(logits, norm(layers[4], "final.norm") @ weights["head"].T)
