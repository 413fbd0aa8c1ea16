"""The Darolix design without a GPU: configuration, registry, tensor names, sizes taken from the tensors, cache needs and
schedule, the command line, and the plain implementation's mechanisms against closed forms (so that the oracle the GPU tests
use is itself pinned)."""
import json
import math

import pytest
import torch

import plain_darolix as plain
from darolix_util import CONFIGS, RANKS, config, make_weights, mamba2, moe, tensor_shapes, write_folder


@pytest.mark.parametrize("name", list(CONFIGS))
def test_config_registry_and_tensor_names(name, tmp_path):
    from tessweave_engine_amd.config import build_model, config_from_dict, read_model_config
    from tessweave_engine_amd.weights.loader import tensor_shapes as stored_shapes
    c = CONFIGS[name]
    config_ = config_from_dict(c)
    assert config_.architecture == "Darolix" and config_.vocab_size == c["vocab"]
    assert config_from_dict(config_.to_dict()) == config_
    folder = write_folder(tmp_path, c, make_weights(c, 0, RANKS[name]))
    assert read_model_config(folder) == config_
    for sized, rank in ((config_, 16), (config_.with_tensor_shapes(stored_shapes(folder)), RANKS[name])):
        specs = {s.name: s.shape for s in build_model(sized).tensor_specs()}
        assert specs == tensor_shapes(c, rank)


def test_a_checkpoint_gives_the_decays_rank_and_must_agree_with_itself(tmp_path):
    from tessweave_engine_amd.weights import WeightError, load_model
    c = CONFIGS["one"]
    weights = make_weights(c, 0, 3)
    model = load_model(write_folder(tmp_path / "a", c, weights), dtype="float32", device="cpu")
    assert model.blocks[0].mixer.branches[1].rank == 3
    weights["l0.mix.right.a2"] = torch.zeros(18, 4, dtype=torch.bfloat16)
    with pytest.raises(WeightError, match="l0.mix.right.a2"):
        load_model(write_folder(tmp_path / "b", c, weights), dtype="float32", device="cpu")
    del weights["l0.mix.right.a1"]
    with pytest.raises(WeightError, match="missing .*l0.mix.right.a1"):
        load_model(write_folder(tmp_path / "c", c, weights), dtype="float32", device="cpu")


def test_config_rejections():
    from tessweave_engine_amd.config import ConfigError, config_from_dict
    base = json.loads(json.dumps(CONFIGS["odd"]))
    for change in (lambda c: c["layers"][0].__setitem__("type", "other"),
                   lambda c: c["layers"][0]["mixer"].pop("right"),
                   lambda c: c["layers"][0]["mixer"]["left"].__setitem__("kv_heads", 4),
                   lambda c: c["layers"][0]["mixer"]["left"].__setitem__("dim", 300),
                   lambda c: c["layers"][0]["mixer"]["left"].pop("scale"),
                   lambda c: c["layers"][0]["mixer"]["left"].__setitem__("softcap", -1.0),
                   lambda c: c["layers"][0]["mixer"]["left"]["q_temp"].__setitem__("every", 0),
                   lambda c: c["layers"][0]["mixer"]["right"].__setitem__("tau", 0),
                   lambda c: c["layers"][0]["mixer"]["right"].__setitem__("dim", 257),
                   lambda c: c["layers"][0]["mlp"].__setitem__("kind", "dense"),
                   lambda c: c["layers"][0]["mlp"]["router"].__setitem__("top", 8),
                   lambda c: c["layers"][0]["mlp"]["router"].__setitem__("identity", -1),
                   lambda c: c["layers"][1]["mixer"].__setitem__("groups", 4),
                   lambda c: c["layers"][1]["mixer"].__setitem__("norm_groups", 7),
                   lambda c: c["layers"][1]["mixer"].__setitem__("conv", 0),
                   lambda c: c["layers"][1]["mixer"].__setitem__("conv", 9),
                   lambda c: c["layers"][1]["mixer"].__setitem__("state", 300),
                   lambda c: c["loop"].__setitem__("stop", 5),
                   lambda c: c["loop"].__setitem__("times", 0),
                   lambda c: c.pop("embedding"),
                   lambda c: c["norm"].__setitem__("eps", 0)):
        c = json.loads(json.dumps(base))
        change(c)
        with pytest.raises(ConfigError):
            config_from_dict(c)


def test_cache_layout_and_schedule():
    """Every run of a layer has a cache slot of its own; each pass of the loop but the first begins with the embedding's
    output added; parallel layers page keys and values and hold the linear attention's state, state-space layers hold
    theirs and the convolution's last inputs."""
    from tessweave_engine_amd.config import build_model, config_from_dict
    model = build_model(config_from_dict(CONFIGS["odd"]))
    assert [(r.block, r.cache_slot, r.adds_embedding) for r in model.schedule] == \
        [(0, 0, False), (1, 1, False), (2, 2, False), (1, 3, True), (2, 4, False), (1, 5, True), (2, 6, False), (3, 7, False)]
    assert model.embedding.keep and model.graph_safe_model
    layout = model.cache_layout()
    a = layout.needs[0].paged
    assert (a.kv_heads, a.head_dim, a.value_dim, a.window) == (3, 32, None, None)
    assert dict(layout.needs[0].states)["linear_attention.s"].shape == (3, 32, 32)
    assert (layout.needs[2].paged.kv_heads, layout.needs[2].paged.head_dim) == (1, 48) and layout.needs[4] == layout.needs[2]
    states = dict(layout.needs[1].states)
    assert layout.needs[1].paged is None and states["state_space.s"].shape == (6, 16, 32)
    assert states["state_space.conv"].shape == (2, 2, 60 + 2 * 6 * 21)
    assert not layout.shares_prefixes
    one = build_model(config_from_dict(CONFIGS["one"]))
    assert [r.block for r in one.schedule] == [0] and not one.embedding.keep
    wide = build_model(config_from_dict(CONFIGS["wide"]))
    assert [(r.block, r.adds_embedding) for r in wide.schedule] == [(0, False), (1, False), (2, False), (0, True), (1, False), (2, False)]


def test_random_weights_and_inspect_on_the_command_line(tmp_path, capsys):
    from tessweave_engine_amd.cli import main
    from tessweave_engine_amd.config import read_model_config
    source = tmp_path / "config.json"
    source.write_text(json.dumps(CONFIGS["wide"]))
    folder = tmp_path / "model"
    assert main(["random-weights", str(source), str(folder), "--seed", "3"]) == 0
    assert read_model_config(folder).to_dict()["layers"] == CONFIGS["wide"]["layers"]
    from safetensors import safe_open
    with safe_open(str(folder / "model.safetensors"), framework="pt") as f:
        assert {k: tuple(f.get_slice(k).get_shape()) for k in f.keys()} == tensor_shapes(CONFIGS["wide"])
    capsys.readouterr()
    assert main(["inspect", str(folder), "--kv-blocks", "10", "--block-size", "16"]) == 0
    assert "Darolix" in capsys.readouterr().out


# ---- the plain implementation's mechanisms against closed forms --------------------------------------------

F64 = torch.float64


def test_sinusoids_and_embedding():
    s = plain.sinusoids(4, 5, F64, start=1000)
    for t, p in enumerate(range(1000, 1004)):
        want = [math.sin(p), math.cos(p), math.sin(p * 10000 ** -0.4), math.cos(p * 10000 ** -0.4), math.sin(p * 10000 ** -0.8)]
        assert torch.allclose(s[t], torch.tensor(want, dtype=F64))
    table = torch.tensor([[1.0, 2.0], [3.0, 4.0]], dtype=F64)
    x = plain.embed([1, 0], table, 3.0)
    assert torch.allclose(x, torch.tensor([[9.0, 13.0], [3.0 + math.sin(1), 6.0 + math.cos(1)]], dtype=F64))


def test_state_space_closed_form():
    """Constant step sizes: the state is a geometric sum; the skip adds D x; heads in a row share a group; the gate comes
    before the norm, which takes the row in equal parts."""
    T, E, N = 5, 2, 3
    g = torch.Generator().manual_seed(0)
    x, B, C = torch.randn(T, E, generator=g, dtype=F64), torch.randn(T, N, generator=g, dtype=F64), torch.randn(T, N, generator=g, dtype=F64)
    dt, log_rate = torch.full((T,), 0.7, dtype=F64), torch.tensor(0.3, dtype=F64)
    y = plain.state_space_steps(x, B, C, dt, log_rate, 1.5)
    decay = math.exp(-math.exp(0.3) * 0.7)
    for t in range(T):
        want = 1.5 * x[t] + sum(decay ** (t - j) * 0.7 * (B[j] @ C[t]) * x[j] for j in range(t + 1))
        assert torch.allclose(y[t], want)
    u = torch.tensor([[3.0, 4.0, 0.0, 2.0]], dtype=F64)
    w = torch.tensor([1.0, 2.0, 3.0, 4.0], dtype=F64)
    n = plain.grouped_rms_norm(u, w, 2, 0.0)
    assert torch.allclose(n, torch.tensor([[3 / math.sqrt(12.5), 8 / math.sqrt(12.5), 0.0, 8 / math.sqrt(2.0)]], dtype=F64))
    assert torch.allclose(plain.softplus(torch.tensor([-1.0, 0.0, 50.0], dtype=F64)),
                          torch.tensor([math.log1p(math.exp(-1)), math.log(2), 50.0], dtype=F64))


def test_state_space_layout_and_convolution():
    """[z | x | B | C | dt] of the packed rows; one convolution with bias and SiLU over x, B and C; two groups of two heads."""
    m = {"heads": 4, "vdim": 1, "state": 2, "groups": 2, "conv": 2, "norm_groups": 1}
    g = torch.Generator().manual_seed(3)
    C, T, width, ch = 3, 4, 4 + 12 + 4, 12
    w = {"in": torch.randn(width, C, generator=g, dtype=F64), "conv": torch.randn(ch, 2, generator=g, dtype=F64),
         "conv.b": torch.randn(ch, generator=g, dtype=F64), "dt_bias": torch.randn(4, generator=g, dtype=F64),
         "A_log": torch.randn(4, generator=g, dtype=F64), "D": torch.randn(4, generator=g, dtype=F64),
         "norm": torch.ones(4, dtype=F64), "o": torch.eye(4, dtype=F64)}
    h = torch.randn(T, C, generator=g, dtype=F64)
    p = h @ w["in"].T
    raw = p[:, 4:16]
    conv = torch.stack([raw[t] * w["conv"][:, 1] + (raw[t - 1] if t else 0) * w["conv"][:, 0] + w["conv.b"] for t in range(T)])
    conv = plain.silu(conv)
    y = torch.zeros(T, 4, dtype=F64)
    for a in range(4):
        k = a // 2
        B, Cc = conv[:, 4 + 2 * k:6 + 2 * k], conv[:, 8 + 2 * k:10 + 2 * k]
        dt = plain.softplus(p[:, 16 + a] + w["dt_bias"][a])
        y[:, a] = plain.state_space_steps(conv[:, a:a + 1], B, Cc, dt, w["A_log"][a], w["D"][a])[:, 0]
    want = plain.rms_unit(y * plain.silu(p[:, :4]), 1e-5)
    assert torch.allclose(plain.mamba2(h, w, m, 1e-5), want)


def test_normed_attention_closed_forms():
    """Keys that are all alike: uniform weights, whatever the scale. The temperature's steps. The cap bounds a score: with a
    huge scale the weights of a matching and an opposed key are as exp(cap) to exp(-cap)."""
    t = plain.query_temperature(10, 0.5, 4)
    assert t.tolist() == [1.0] * 3 + [1 + 0.5 * math.log(2)] * 4 + [1 + 0.5 * math.log(3)] * 3
    T, C = 5, 3
    g = torch.Generator().manual_seed(1)
    h = torch.randn(T, C, generator=g, dtype=F64)
    m = {"heads": 2, "kv_heads": 1, "dim": 2, "vdim": 3, "scale": 2.0, "softcap": 3.0, "q_temp": {"coef": 0.3, "every": 2}}
    w = {"q": torch.randn(4, C, generator=g, dtype=F64), "k": torch.zeros(2, C, dtype=F64), "v": torch.randn(3, C, generator=g, dtype=F64),
         "o": torch.randn(C, 6, generator=g, dtype=F64)}
    mean = torch.cumsum(h @ w["v"].T, 0) / torch.arange(1, T + 1, dtype=F64).view(-1, 1)
    assert torch.allclose(plain.normed_attention(h, w, m, 1e-5), torch.cat([mean, mean], 1) @ w["o"].T)
    h = torch.tensor([[1.0, 0.0], [-1.0, 1.0]], dtype=F64)
    m = {"heads": 1, "kv_heads": 1, "dim": 1, "vdim": 1, "scale": 1e6, "softcap": 2.0}
    w = {"q": torch.tensor([[1.0, 0.0]], dtype=F64), "k": torch.tensor([[1.0, 0.0]], dtype=F64),
         "v": torch.tensor([[0.0, 1.0]], dtype=F64), "o": torch.tensor([[1.0], [0.0]], dtype=F64)}
    want = math.exp(2) / (math.exp(2) + math.exp(-2))
    assert torch.allclose(plain.normed_attention(h, w, m, 1e-9)[:, 0], torch.tensor([0.0, want], dtype=F64))


def test_gated_linear_attention_closed_form():
    """Constant decays per key element: o_t = sum_j sum_d q_td a_d^(t - j) k_jd v_j. The decay is a root of a sigmoid."""
    T, D, E = 5, 3, 2
    g = torch.Generator().manual_seed(5)
    q, k, v = (torch.randn(T, n, generator=g, dtype=F64) for n in (D, D, E))
    a = torch.tensor([0.9, 0.5, 1.0], dtype=F64)
    o = plain.linear_attention_steps(q, k, v, a.expand(T, D))
    for t in range(T):
        want = sum((q[t] * a ** (t - j) * k[j]).sum() * v[j] for j in range(t + 1))
        assert torch.allclose(o[t], want)
    m = {"heads": 1, "dim": 1, "vdim": 1, "tau": 4.0}
    one, zero = torch.ones(1, 1, dtype=F64), torch.zeros(1, 1, dtype=F64)
    w = {"q": one, "k": one, "v": one, "g": one, "a1": one, "a2": one, "a2.b": torch.tensor([0.5], dtype=F64),
         "norm": torch.ones(1, dtype=F64), "o": one}
    h = torch.tensor([[1.0], [2.0]], dtype=F64)
    alpha = (1 / (1 + math.exp(-2.5))) ** 0.25
    s = alpha * 1.0 + 4.0                                          # the state at the second token, times q = 2
    want = (2 * s) / math.sqrt((2 * s) ** 2 + 1e-5) * (2 / (1 + math.exp(-2)))
    assert torch.allclose(plain.gated_linear_attention(h, w, m, 1e-5)[1, 0], torch.tensor(want, dtype=F64))
    assert torch.allclose(plain.gated_linear_attention(h, dict(w, g=zero), m, 1e-5), torch.zeros(2, 1, dtype=F64))


def test_experts_closed_forms():
    """Scores are a softmax over all experts; the correction decides the choice and does not weigh; the chosen scores are
    made to sum to one; an identity expert returns its input."""
    C = 3
    g = torch.Generator().manual_seed(1)
    w = {"router": torch.diag(torch.tensor([1.0, 2.0, 3.0], dtype=F64)), "correction": torch.tensor([0.9, 0.0, 0.0], dtype=F64)}
    for e in range(2):
        w[f"e{e}.gate"], w[f"e{e}.up"] = (torch.randn(4, C, generator=g, dtype=F64) for _ in range(2))
        w[f"e{e}.down"] = torch.randn(C, 4, generator=g, dtype=F64)
    h = torch.tensor([[0.1, 0.5, 1.0]], dtype=F64)
    s = torch.softmax(torch.tensor([0.1, 1.0, 3.0], dtype=F64), 0)
    mlp = {"router": {"experts": 2, "identity": 1, "top": 2}, "expert": {"ff": 4}}
    e0 = plain.expert(h, w["e0.gate"], w["e0.up"], w["e0.down"])
    want = (s[0] * e0 + s[2] * h) / (s[0] + s[2])                  # the first is chosen for its correction
    assert torch.allclose(plain.routed_ff(h, w, mlp), want)
    w["correction"] = torch.zeros(3, dtype=F64)
    e1 = plain.expert(h, w["e1.gate"], w["e1.up"], w["e1.down"])
    assert torch.allclose(plain.routed_ff(h, w, mlp), (s[1] * e1 + s[2] * h) / (s[1] + s[2]))
    z = h @ w["e0.gate"].T
    assert torch.allclose(e0, ((z / (1 + torch.exp(-z))) * (h @ w["e0.up"].T)) @ w["e0.down"].T)


def test_layer_arrangement_and_loop():
    """One norm, both sublayers read its result; the looped layers run again behind the embedding's output added once; half
    of each normed result in a parallel layer."""
    c = CONFIGS["odd"]
    weights = {k: v.double() for k, v in make_weights(c, 2, RANKS["odd"]).items()}
    toks = [3, 50, 7, 7, 90, 1, 200, 4]
    layers = []
    logits = plain.forward(c, weights, toks, layers_out=layers)
    assert len(layers) == 8 and plain.layer_runs(c) == [(0, False), (1, False), (2, False), (1, True), (2, False), (1, True), (2, False), (3, False)]
    eps = c["norm"]["eps"]
    first = plain.embed(toks, weights["embed"], c["embedding"]["scale"])
    h = plain.rms_norm(first, weights["l0.norm1"], eps)
    m = c["layers"][0]["mixer"]
    left = plain.normed_attention(h, plain.sub(weights, "l0.mix.left."), m["left"], eps)
    right = plain.gated_linear_attention(h, plain.sub(weights, "l0.mix.right."), m["right"], eps)
    y = 0.5 * plain.rms_norm(left, weights["l0.mix.left.out"], eps) + 0.5 * plain.rms_norm(right, weights["l0.mix.right.out"], eps)
    y = y + plain.routed_ff(h, plain.sub(weights, "l0.mlp."), c["layers"][0]["mlp"])
    assert torch.allclose(layers[0], first + y)
    x = layers[2] + first
    h = plain.rms_norm(x, weights["l1.norm1"], eps)
    y = plain.mamba2(h, plain.sub(weights, "l1.mix."), c["layers"][1]["mixer"], eps) + \
        plain.routed_ff(h, plain.sub(weights, "l1.mlp."), c["layers"][1]["mlp"])
    assert torch.allclose(layers[3], x + y)
    h = plain.rms_norm(layers[6], weights["l3.norm1"], eps)
    assert torch.allclose(layers[7], layers[6] + plain.mamba2(h, plain.sub(weights, "l3.mix."), c["layers"][3]["mixer"], eps))
    assert torch.allclose(logits, plain.rms_norm(layers[7], weights["final.norm"], eps) @ weights["head"].T)
    single = config([mamba2(2, 4, 4, 1, 2, 2, mlp=moe(2, 1, 1, 8))], width=12, vocab=20)
    assert plain.layer_runs(single) == [(0, False)]
