"""The Vulosun design on the GPU against the plain implementation (`plain_vulosun.py`).

Mechanisms alone (each kernel against the plain function of the same mechanism: layer norms of results and stream, queries
and keys normed by the row or the head, turned both ways, the maps of differential heads, attention made sharp so that one
key among hundreds carries the row, in chunks, with sinks and gates, the combined maps, lightning attention's states walked, in
chunks and in segments over cut sequences in reused slots, the gated norm behind it, the router's groups, the plain experts
left apart), then each mixer and feed-forward alone in a model of one or two layers, then whole models through the package's
loader, cache manager and step function: prefill against token-by-token decoding, portions down to two tokens, unequal
batches against each request alone, few pages and slots that are freed and used again, keys just inside and just outside
every chunk, a long prompt, a state that must survive hundreds of tokens, long decoding from HIP graphs, sizes drawn at random,
and greedy generation through the scheduler.

Bars: float32 rows must agree with the float64 plain implementation to 2e-5 of the logits' spread (the kernels sum in other
orders) plus three times what the PLAIN implementation run in float32 is off by in that row. bfloat16 rows must agree to 3 %
of the spread, one in five up to three times as far (the narrow models here round coarsely). A token whose expert or group
scores nearly tie (`plain.choose_experts`' margin under CLOSE) may go the other way in bfloat16, and what it leaves in states
and caches reaches every later row of its sequence: rows behind a sequence's first such token are only held to a typical
error within five times the bar. Every kernel that runs in bfloat16 is the same template as in float32.
"""
import math
import random

import numpy as np
import pytest
import torch

import plain_vulosun as plain
from vulosun_util import (CONFIGS, Driver, attention, config, dense, differential, left, make_weights, moe, parallel, right, rot,
                          row_error, write_folder)

pytestmark = pytest.mark.gpu

BAR = {"float32": 2e-5, "bfloat16": 3e-2}
CLOSE = 0.02         # a margin of scores under this may go the other way in bfloat16
LENGTHS = {"odd": (61, 23, 9, 150, 1), "wide": (70, 12, 33, 101, 2), "one": (40, 7, 90)}


def double(weights):
    return {k: v.double() for k, v in weights.items()}


class Slack(np.ndarray):
    """Router margins per row that also carry, as `.float32`, what the plain implementation in float32 is off by."""


def reference(c, weights, toks):
    """(logits [T, V] in float64, per token the smallest router margin with the float32 slack per row on it)."""
    margins = []
    logits = plain.forward(c, double(weights), toks, margins=margins).numpy()
    least = torch.stack(margins).min(0).values.numpy() if margins else np.full(len(toks), np.inf)
    least = np.asarray(least, dtype=np.float64).view(Slack)
    single = plain.forward(c, {k: v.float() for k, v in weights.items()}, toks, dtype=torch.float32).numpy()
    least.float32 = row_error(single, logits)
    return logits, least


def tdtype(name):
    return getattr(torch, name)


def ints(values, device):
    return torch.tensor(values, dtype=torch.int32, device=device)


# ---------------------------------------------------------------------------------------------------------
# mechanisms alone

@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("C", [50, 88, 4, 1000, 2048, 5000, 9000])
def test_layer_norms_of_a_result_and_the_stream(device, dtype, C):
    """A result from rows, from split-K sums, from experts' rows and from both; with and without norms of either; a stream
    whose mean is far from zero; chosen rows only; row lengths of every kind (whole vectors or not, one and several pieces a thread)."""
    from tessweave_engine_amd.kernels import ops
    g = torch.Generator().manual_seed(C)
    n, eps, top = 7, 1e-5, 3
    x = 5.0 * torch.randn(n, C, generator=g) + 40.0
    y, parts = 3.0 * torch.randn(n, C + 4, generator=g) - 7.0, torch.randn(5, n, C, generator=g)
    pair_rows, weights = torch.randn(30, C, generator=g), torch.rand(n, top, generator=g)
    pos = torch.randint(0, 30, (n * top,), generator=g).to(torch.int32)
    pos[4] = -1                                                     # (a choice without a row adds nothing)
    (w1, b1), (w2, b2) = ((1.0 + 0.3 * torch.randn(C, generator=g), torch.randn(C, generator=g)) for _ in range(2))
    chosen = pair_rows.double()[pos.long()].view(n, top, C) * weights.double().unsqueeze(-1)
    chosen[4 // top, 4 % top] = 0.0
    to = lambda t: t.to(device).contiguous()                        # noqa: E731
    results = {"rows": (dict(y=to(y)[:, :C]), y[:, :C].double()), "sums": (dict(add=to(parts)), parts.double().sum(0)),
               "experts": (dict(pairs=(to(pair_rows), to(pos), to(weights))), chosen.sum(1)),
               "both": (dict(add=to(parts), pairs=(to(pair_rows), to(pos), to(weights))), parts.double().sum(0) + chosen.sum(1)),
               "rows and experts": (dict(y=to(y)[:, :C], pairs=(to(pair_rows), to(pos), to(weights))), y[:, :C].double() + chosen.sum(1))}
    tol = 1e-5 if dtype == "float32" else 2e-2
    for what, (given, result) in results.items():
        for post in (True, False):
            got, out = x.to(device), torch.full((n, C), float("nan"), dtype=tdtype(dtype), device=device)
            ops.layer_norm(got, eps, post=(to(w1), to(b1)) if post else None, norm=(to(w2), to(b2)), out=out, **given)
            want = x.double() + (plain.layer_norm(result, w1.double(), b1.double(), eps) if post else result)
            assert torch.allclose(got.double().cpu(), want, atol=2e-5, rtol=1e-6), (what, post)
            assert torch.allclose(out.double().cpu(), plain.layer_norm(want, w2.double(), b2.double(), eps), atol=3 * tol, rtol=tol), (what, post)
    got = x.to(device)
    ops.layer_norm(got, eps, post=(to(w1), to(b1)), **results["sums"][0])              # nobody reads the stream
    assert torch.allclose(got.double().cpu(), x.double() + plain.layer_norm(parts.double().sum(0), w1.double(), b1.double(), eps), atol=2e-5, rtol=1e-6)
    got, out = x.to(device), torch.empty(3, C, dtype=tdtype(dtype), device=device)
    ops.layer_norm(got, eps, norm=(to(w2), to(b2)), out=out, rows=ints([6, 0, 3], device), **results["sums"][0])
    want = plain.layer_norm((x.double() + parts.double().sum(0))[[6, 0, 3]], w2.double(), b2.double(), eps)
    assert torch.equal(got.cpu(), x) and torch.allclose(out.double().cpu(), want, atol=3 * tol, rtol=tol)


def test_exact_rotary_tables_far_out(device):
    from tessweave_engine_amd.parts import RotaryEmbedding, StepContext, Workspace
    for base, dims, factor in ((1e6, 96, 1.0), (50000.0, 8, 4.0), (100.0, 2, 2.5)):
        part = RotaryEmbedding(dims, base, dims, divide=factor)
        part.bind({}, torch.float32, device)
        ctx = StepContext()
        positions = [0, 1, 2, 63, 999, 4097, 30000, 250001]
        ctx.positions, ctx.n_tokens, ctx.max_tokens = ints([positions], device), len(positions), 16
        ctx.workspace = Workspace(device)
        cos, sin = part.tables(ctx)
        a = torch.tensor(positions, dtype=torch.float64).view(-1, 1) * base ** (-2.0 * torch.arange(dims // 2, dtype=torch.float64) / dims) / factor
        assert (cos.double().cpu() - torch.cos(a)).abs().max() < 5e-7 and (sin.double().cpu() - torch.sin(a)).abs().max() < 5e-7


SHARP = [  # H, G, D, E, rotated, page, splits of the projection
    (4, 2, 24, 20, 10, 4, 1), (8, 8, 32, 64, 32, 16, 3), (6, 1, 50, 34, 4, 8, 1), (3, 3, 128, 96, 128, 16, 2), (10, 2, 64, 64, 2, 16, 1),
    (2, 2, 15, 7, 6, 4, 5), (1, 1, 30, 100, 30, 16, 1), (32, 2, 64, 48, 64, 16, 1)]


def sharp_targets(T, page, chunk=None):
    """Per query, the ONE key it is made to point at: the first, one at a page's end or start, its neighbour, itself, one far
    back; with chunks also the chunk's first and the last one outside (which it must not see)."""
    out = []
    for i in range(T):
        lo = i // chunk * chunk if chunk else 0
        options = [0, i // page * page - 1, i // page * page, i - 1, i, i // 2, i - 97] + ([lo, lo - 1, lo, lo + 1] if chunk else [])
        out.append(min(max(options[i % len(options)], 0), i))
    return out


def pages_of(T, page, G, dev, dtype, device):
    """Pages in an order of their own that hold what other requests left: (keys, values, block table, slot per token)."""
    blocks = (T + page - 1) // page
    order = list(range(blocks + 3))
    random.Random(3).shuffle(order)
    table = order[:blocks]
    keys = torch.full((blocks + 3, G, page, dev), 50.0, dtype=dtype, device=device)
    values = torch.full((blocks + 3, G, page, dev), float("nan"), dtype=dtype, device=device)
    slots = ints([table[t // page] * page + t % page for t in range(T)], device)
    return keys, values, ints([table + [-1, -1]], device), slots


def unturned(x, kind, r):
    """x such that rotation by `kind` gives back x (the inverse turn), so that tests can say what the turned rows are."""
    n, half = r["dims"], r["dims"] // 2
    a = -plain.angles(x.shape[0], r, x.dtype).unsqueeze(1)
    if kind == "half":
        u, v = plain.turn(x[..., :half], x[..., half:n], a)
        return torch.cat([u, v, x[..., n:]], -1)
    u, v = plain.turn(x[..., 0:n:2], x[..., 1:n:2], a)
    return torch.cat([torch.stack([u, v], -1).flatten(-2), x[..., n:]], -1)


def split_rows(src, splits, g, device):
    """SRC as it stands, or as split-K sums that add up to it."""
    if splits == 1:
        return src.to(device)
    parts = torch.randn(splits, *src.shape, generator=g)
    parts[0] = src - parts[1:].sum(0)
    return parts.to(device)


def rows_of(parts, lo, hi):
    return parts[lo:hi] if parts.dim() == 2 else parts[:, lo:hi].contiguous()


def run_portions(ops, rows, T, columns, norm, weights, rotation, keys, values, bt, slots, sizes, out, scale, maps, adjacent, device, bias=None,
                 chunk=0, sink=None, gated=True, splits_decode=1, value_scale=1.0):
    """Two prompt portions (the first cut where no page and no chunk ends), then single tokens, through the finishing kernel and
    the attention kernels."""
    H, G, D, E, dev = sizes
    q = torch.empty(T, H * maps * dev, dtype=keys.dtype, device=device)
    for lo, hi in [(0, 37), (37, 170)] + [(t, t + 1) for t in range(170, T)]:
        n = hi - lo
        gate = torch.full((n, H), float("nan"), device=device) if columns[3] is not None else None
        ops.rows_finish(rows_of(rows, lo, hi), columns, norm, *weights, (ints(list(range(lo, hi)), device), *rotation), q[lo:hi], keys, values,
                        slots[lo:hi].contiguous(), gate, H, G, D, E, 1e-5, maps=maps, adjacent=adjacent, bias=bias, value_scale=value_scale)
        starts, lens = ints([0, n], device), ints([hi], device)
        extra = dict(chunk=chunk, sink=sink, gate=gate if gated else None)
        if n > 1:
            split = ops.attn_prefill_split(1, H * maps, G, n, hi)
            ws = torch.empty(max(1, ops.attn_prefill_workspace_floats(n, H * maps, dev, split[0])), device=device) if split[0] > 1 else None
            ops.attn_prefill(q[lo:hi], keys, values, bt, starts, lens, 0, 1, n, out[lo:hi], H * maps, G, dev, scale, split=split, workspace=ws, **extra)
        else:
            ws = torch.empty(ops.attn_decode_workspace_floats(1, H * maps, dev, splits_decode), device=device) if splits_decode > 1 else None
            ops.attn_decode(q[lo:hi], keys, values, bt, starts, lens, 0, 1, out[lo:hi], H * maps, G, dev, scale, splits=splits_decode,
                            workspace=ws, **extra)
        if gate is not None:
            yield lo, hi, gate
    return


def frequencies(r, device):
    """(frequencies, what float32 rounds off them) of a rotation."""
    f = plain.angles(2, r, torch.float64)[1]
    return f.float().to(device), (f - f.float().double()).float().to(device)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("splits_decode", [1, 3])
@pytest.mark.parametrize("H,G,D,E,turned,page,splits", SHARP)
def test_head_norms_rotation_and_sinks_made_sharp(device, dtype, H, G, D, E, turned, page, splits, splits_decode):
    """Norms per head, rotated halves, cache write (values times the branch's weight) and attention with sinks. Every query
    points at ONE key. A key lost or seen wrongly moves its row by the size of a value; a sink lost moves all."""
    from tessweave_engine_amd.kernels import ops
    T, eps, vs = 200, 1e-5, 0.7
    r = rot(300.0, turned)
    scale = 9.0 / D
    g = torch.Generator().manual_seed(H * D + page)
    dev = (max(D, E) + 15) // 16 * 16
    targets = sharp_targets(T, page)
    wq, wk = 1.0 + 0.2 * torch.randn(D, generator=g), 1.0 + 0.2 * torch.randn(D, generator=g)
    k_turned = torch.randn(T, G, D, generator=g, dtype=torch.float64)
    k_turned = k_turned / k_turned.norm(dim=-1, keepdim=True) * math.sqrt(D)
    q_turned = k_turned[targets].repeat_interleave(H // G, 1)
    q = (unturned(q_turned, "half", r) / wq.double()).float() * 3.0
    k = (unturned(k_turned, "half", r) / wk.double()).float() * 0.6
    v = torch.randn(T, G * E, generator=g)
    sink = torch.linspace(2.0, 9.0, H)
    at = [0, (H * D + 3) // 4 * 4]
    at.append(at[1] + (G * D + 3) // 4 * 4)
    src = torch.zeros(T, at[2] + G * E + 1)
    src[:, :H * D], src[:, at[1]:at[1] + G * D], src[:, at[2]:at[2] + G * E] = q.reshape(T, -1), k.reshape(T, -1), v
    m = {"heads": H, "kv_heads": G, "dim": D, "vdim": E, "scale": scale, "rot": r}
    eye = torch.eye(src.shape[1], dtype=torch.float64)
    w = {"q": eye[:H * D], "k": eye[at[1]:at[1] + G * D], "v": eye[at[2]:at[2] + G * E], "o": torch.eye(H * E, dtype=torch.float64),
         "q.norm": wq.double(), "k.norm": wk.double(), "sink": sink.double()}
    want = vs * plain.head_normed_attention(src.double(), w, m, eps)
    dt = tdtype(dtype)
    keys, values, bt, slots = pages_of(T, page, G, dev, dt, device)
    out = torch.full((T, H * dev), float("nan"), dtype=dt, device=device)
    for _ in run_portions(ops, split_rows(src, splits, g, device), T, (0, at[1], at[2], None), "head", (wq.to(device), wk.to(device)), frequencies(r, device),
                          keys, values, bt, slots, (H, G, D, E, dev), out, scale, 1, False, device, sink=sink.to(device),
                          splits_decode=splits_decode, value_scale=vs):
        pass
    got = out.view(T, H, dev).double().cpu()
    err = (got[:, :, :E].reshape(T, H * E) - want).abs().amax(1)
    tol = 1e-4 if dtype == "float32" else 0.12
    assert err.max() < tol, (int(err.argmax()), targets[int(err.argmax())], float(err.max()))
    assert not got[:, :, E:].any()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("splits_decode", [1, 4])
@pytest.mark.parametrize("H,G,D,E,turned,page,splits", SHARP)
def test_row_norms_rotation_and_gates_made_sharp(device, dtype, H, G, D, E, turned, page, splits, splits_decode):
    """Norms over the whole row, rotated neighbours, gates from the same rows, attention whose result carries the gate."""
    from tessweave_engine_amd.kernels import ops
    T, eps = 200, 1e-5
    r = rot(300.0, turned, 1.7)
    scale = 9.0 / D
    g = torch.Generator().manual_seed(H * D + page)
    dev = (max(D, E) + 15) // 16 * 16
    targets = sharp_targets(T, page)
    wq, wk = 1.0 + 0.2 * torch.randn(H * D, generator=g), 1.0 + 0.2 * torch.randn(G * D, generator=g)
    k_turned = torch.randn(T, G, D, generator=g, dtype=torch.float64)
    k_turned = k_turned / k_turned.norm(dim=-1, keepdim=True) * math.sqrt(D)
    q_turned = k_turned[targets].repeat_interleave(H // G, 1)
    q = (unturned(q_turned, "near", r).reshape(T, -1) / wq.double()).float() * 3.0
    k = (unturned(k_turned, "near", r).reshape(T, -1) / wk.double()).float() * 0.6
    v, z = torch.randn(T, G * E, generator=g), 2.0 * torch.randn(T, H, generator=g)
    at = [0, (H * D + 3) // 4 * 4]
    at += [at[1] + (G * D + 3) // 4 * 4]
    at += [at[2] + (G * E + 3) // 4 * 4]
    src = torch.zeros(T, at[3] + H)
    src[:, :H * D], src[:, at[1]:at[1] + G * D], src[:, at[2]:at[2] + G * E], src[:, at[3]:] = q, k, v, z
    m = {"heads": H, "kv_heads": G, "dim": D, "vdim": E, "scale": scale, "rot": r}
    eye = torch.eye(src.shape[1], dtype=torch.float64)
    w = {"q": eye[:H * D], "k": eye[at[1]:at[1] + G * D], "v": eye[at[2]:at[2] + G * E], "g": eye[at[3]:], "o": torch.eye(H * E, dtype=torch.float64),
         "q.norm": wq.double(), "k.norm": wk.double()}
    want = plain.whole_normed_attention(src.double(), w, m, eps)
    dt = tdtype(dtype)
    keys, values, bt, slots = pages_of(T, page, G, dev, dt, device)
    out = torch.full((T, H * dev), float("nan"), dtype=dt, device=device)
    for lo, hi, gate in run_portions(ops, split_rows(src, splits, g, device), T, (0, *at[1:]), "row", (wq.to(device), wk.to(device)), frequencies(r, device),
                                     keys, values, bt, slots, (H, G, D, E, dev), out, scale, 1, True, device, splits_decode=splits_decode):
        assert torch.allclose(gate.double().cpu(), torch.sigmoid(z[lo:hi].double()), atol=1e-6)
    err = (out.view(T, H, dev)[:, :, :E].double().cpu().reshape(T, H * E) - want).abs().amax(1)
    tol = 1e-4 if dtype == "float32" else 0.12
    assert err.max() < tol, (int(err.argmax()), targets[int(err.argmax())], float(err.max()))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("chunk,splits_decode", [(1, 1), (7, 1), (16, 2), (64, 1), (50, 3), (128, 2), (1000, 1)])
@pytest.mark.parametrize("H,G,D,E,turned,page,splits", [(4, 2, 24, 20, 10, 4, 1), (3, 3, 32, 64, 8, 16, 3), (12, 1, 15, 34, 2, 8, 1), (2, 1, 64, 128, 64, 16, 2),
                                                        (6, 3, 11, 7, 6, 4, 1), (16, 2, 100, 200, 40, 16, 1)])
def test_differential_maps_in_chunks_made_sharp(device, dtype, chunk, splits_decode, H, G, D, E, turned, page, splits):
    """Both maps' scores against the same values, in chunks counted from the sequence's start, and the maps combined. Each map's
    query points at a key of its own: the chunk's first, the last one outside, one far back, itself."""
    from tessweave_engine_amd.kernels import ops
    T, eps, diff = 200, 1e-5, 0.35
    r = rot(200.0, turned, 2.0)
    scale = 14.0 / D
    g = torch.Generator().manual_seed(H * D + chunk)
    dev = (max(2 * D, E) + 15) // 16 * 16
    targets = sharp_targets(T, page, chunk)
    k_turned = torch.randn(T, G, 2, D, generator=g, dtype=torch.float64)
    k_turned = k_turned / k_turned.norm(dim=-1, keepdim=True) * math.sqrt(D)
    other = [t // 2 for t in targets]
    q_turned = torch.stack([k_turned[targets][:, :, 0], k_turned[other][:, :, 1]], 2).repeat_interleave(H // G, 1)
    turn_back = lambda x, heads: unturned(x.reshape(T, heads * 2, D), "near", r).reshape(T, -1)          # noqa: E731
    bias = 0.5 * torch.randn(2 * (H + G) * D + G * E + H + 8, generator=g)
    at = [0, (H * 2 * D + 3) // 4 * 4]
    at += [at[1] + (G * 2 * D + 3) // 4 * 4]
    at += [at[2] + (G * E + 3) // 4 * 4]
    bias = bias[:at[3] + H].contiguous()
    bias[at[3]:] = 0.0                                                # (the gates have none)
    z = torch.randn(T, H, generator=g)
    src = torch.zeros(T, at[3] + H)
    src[:, :H * 2 * D] = turn_back(q_turned, H).float() - bias[:H * 2 * D]
    src[:, at[1]:at[1] + G * 2 * D] = turn_back(k_turned, G).float() - bias[at[1]:at[1] + G * 2 * D]
    src[:, at[2]:at[2] + G * E], src[:, at[3]:] = torch.randn(T, G * E, generator=g), z
    lam = [0.4 * torch.randn(D, generator=g, dtype=torch.float64) for _ in range(4)]
    m = {"heads": H, "kv_heads": G, "dim": D, "vdim": E, "scale": scale, "rot": r, "mask": {"size": chunk}, "diff": diff}
    eye = torch.eye(src.shape[1], dtype=torch.float64)
    w = {"g": eye[at[3]:], "o": torch.eye(H * E, dtype=torch.float64), **dict(zip(("lq1", "lk1", "lq2", "lk2"), lam))}
    for name, lo, rows in (("q", 0, H * 2 * D), ("k", at[1], G * 2 * D), ("v", at[2], G * E)):
        w[name], w[name + ".b"] = eye[lo:lo + rows], bias[lo:lo + rows].double()
    want = plain.differential_attention(src.double(), w, m, eps)
    weight = float(plain.differential_lambda(w, diff))
    dt = tdtype(dtype)
    keys, values, bt, slots = pages_of(T, page, G, dev, dt, device)
    maps = torch.full((T, 2 * H * dev), float("nan"), device=device)
    out = torch.full((T, H * ((E + 7) // 8 * 8)), float("nan"), dtype=dt, device=device)
    rows = split_rows(src, splits, g, device)
    for lo, hi, gate in run_portions(ops, rows, T, (0, *at[1:]), None, (None, None), frequencies(r, device), keys, values, bt, slots,
                                     (H, G, D, E, dev), maps, scale, 2, True, device, bias=bias.to(device), chunk=chunk, gated=False,
                                     splits_decode=splits_decode):
        ops.map_difference(maps[lo:hi], out[lo:hi], H, E, weight, 1.0 - diff, eps, gate=gate)
    got = out.view(T, H, -1).double().cpu()
    # where a map's difference is nearly nothing its norm blows rounding up: held to what float32 or bfloat16 leaves of it
    k_plain, v_plain = plain.chunked_keys_values(src.double(), w, m)
    q_plain = plain.rotate_neighbours((src.double() @ w["q"].T + w["q.b"]).view(T, 2 * H, D), r).view(T, H, 2, D)
    a1, a2 = (plain.attend(q_plain[:, :, i], k_plain[:, :, i], v_plain, scale, plain.same_chunk(T, chunk)) for i in (0, 1))
    size = (a1 - weight * a2).pow(2).mean(-1).sqrt().clamp(max=1.0)
    err = ((got[:, :, :E] - want.view(T, H, E)).abs().amax(-1) * size).amax(1)
    tol = 1e-4 if dtype == "float32" else 0.12
    assert err.max() < tol, (int(err.argmax()), targets[int(err.argmax())], float(err.max()))
    assert not got[:, :, E:].any()
    # a layer that reads these pages with queries alone: the same rows, none written
    before = keys.clone(), values.nan_to_num().clone()
    q = torch.empty(T, H * 2 * dev, dtype=dt, device=device)
    gate = torch.empty(T, H, device=device)
    ops.rows_finish(rows, (0, None, None, at[3]), None, None, None, (ints(list(range(T)), device), *frequencies(r, device)), q, keys, values, slots, gate, H, G, D, E, eps, maps=2, adjacent=True,
                    bias=bias.to(device))
    assert torch.equal(keys, before[0]) and torch.equal(values.nan_to_num(), before[1])
    ops.attn_prefill(q, keys, values, bt, ints([0, T], device), ints([T], device), 0, 1, T, maps, 2 * H, G, dev, scale, chunk=chunk)
    ops.map_difference(maps, out, H, E, weight, 1.0 - diff, eps, gate=gate)
    err = ((out.view(T, H, -1)[:, :, :E].double().cpu() - want.view(T, H, E)).abs().amax(-1) * size).amax(1)
    assert err.max() < tol


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("chunk", [32, 300, 700])
def test_chunks_over_long_keys_and_split_tiles(device, dtype, chunk):
    """900 tokens behind 500: tiles of rows whose keys are cut for several workgroups, tiles that straddle a chunk's edge, with
    sinks and gates; the same tokens one by one with keys cut into ranges."""
    from tessweave_engine_amd.kernels import ops
    T, H, G, D, page = 1400, 4, 2, 64, 16
    g = torch.Generator().manual_seed(chunk)
    q, k, v = (torch.randn(T, n, D, generator=g) for n in (H, G, G))
    q = 3.0 * q
    dt = tdtype(dtype)
    sink, gate = torch.randn(H, generator=g), torch.rand(T, H, generator=g)
    rounded = [t.to(dt).double() for t in (q, k, v)]
    want = plain.attend(*rounded, 0.125, plain.same_chunk(T, chunk), sink.double()) * gate.double().unsqueeze(-1)
    keys, values, bt, slots = pages_of(T, page, G, D, dt, device)
    at = slots.long()
    keys[at // page, :, at % page] = k.to(device).to(dt)
    v_pages = values.view(values.shape[0], G, D, page)
    v_pages[at // page, :, :, at % page] = v.to(device).to(dt)
    v_pages.nan_to_num_(50.0)
    qd = q.to(device).to(dt).view(T, H * D)
    out = torch.full((T, H * D), float("nan"), device=device)
    for lo, hi in ((0, 500), (500, 1400)):
        n = hi - lo
        for split in (ops.attn_prefill_split(1, H, G, n, min(hi, chunk + 128)), ops.attn_prefill_split(1, H, G, n, hi), (1, 0, 64)):
            ws = torch.full((max(1, ops.attn_prefill_workspace_floats(n, H, D, split[0])),), float("nan"), device=device)
            ops.attn_prefill(qd[lo:hi], keys, values, bt, ints([0, n], device), ints([hi], device), 0, 1, n, out[lo:hi], H, G, D, 0.125, split=split,
                             workspace=ws, chunk=chunk, sink=sink.to(device), gate=gate[lo:hi].to(device).contiguous())
            assert (out[lo:hi].view(n, H, D).double().cpu() - want[lo:hi]).abs().max() < (2e-5 if dtype == "float32" else 3e-2), (lo, split)
    for t in (0, 31, 32, 299, 300, 301, 698, 700, 1399):
        for splits in (1, 2, 5):
            one = torch.full((1, H * D), float("nan"), device=device)
            ws = torch.full((max(1, ops.attn_decode_workspace_floats(1, H, D, splits)),), float("nan"), device=device)
            ops.attn_decode(qd[t:t + 1], keys, values, bt, ints([0, 1], device), ints([t + 1], device), 0, 1, one, H, G, D, 0.125, splits=splits,
                            workspace=ws, chunk=chunk, sink=sink.to(device), gate=gate[t:t + 1].to(device).contiguous())
            assert (one.view(H, D).double().cpu() - want[t]).abs().max() < (2e-5 if dtype == "float32" else 3e-2), (t, splits)


def lightning_rows(H, D, E, T, decay, seed):
    g = torch.Generator().manual_seed(seed)
    rows = torch.randn(T, 2 * H * D + H * E, generator=g)
    act = plain.silu(rows.double())
    q, k, v = act[:, :H * D].view(T, H, D), act[:, H * D:2 * H * D].view(T, H, D), act[:, 2 * H * D:].view(T, H, E)
    return rows, torch.stack([plain.lightning_steps(q[:, a], k[:, a], v[:, a], decay[a]) for a in range(H)], 1).reshape(T, H * E)


@pytest.mark.parametrize("walk", [True, False], ids=["walked", "chunks"])
@pytest.mark.parametrize("H,D,E", [(3, 20, 24), (1, 13, 10), (4, 128, 64), (2, 256, 16), (2, 64, 200), (4, 100, 7), (8, 12, 70)])
def test_lightning_states_over_cut_sequences_in_reused_slots(device, H, D, E, walk):
    """Three sequences cut differently (one whole, one in portions of 1, 2, 5 and 33 tokens, one token by token), their
    states in slots that other sequences used before; decays from one to almost nothing."""
    from tessweave_engine_amd.kernels import ops
    Dp, Ep = (D + 15) // 16 * 16, (E + 15) // 16 * 16
    decay = [1.0, 0.999, 0.6, 1e-6, 0.9, 0.05, 0.3, 0.99][:H]
    cuts = [[170], [1, 2, 5, 33, 1, 2, 5, 10], [1] * 23]
    cases = [lightning_rows(H, D, E, sum(cut), decay, H * D + s) for s, cut in enumerate(cuts)]
    state = torch.randn(4, H, Ep, Dp, device=device)
    slots = [2, 0, 3]
    untouched = state[1].clone()
    for s in slots:
        state[s].zero_()
    at = [0, 0, 0]
    outs = [torch.zeros(sum(cut), H * E, device=device) for cut in cuts]
    while any(cuts):
        rows, q_start, sl, who = [], [0], [], []
        for s in range(3):
            if cuts[s]:
                n = cuts[s].pop(0)
                rows.append(cases[s][0][at[s]:at[s] + n])
                q_start.append(q_start[-1] + n)
                sl.append(slots[s])
                who.append((s, at[s], n))
                at[s] += n
        src = torch.cat(rows).contiguous().to(device)
        out = torch.full((src.shape[0], H * E), float("nan"), device=device)
        longest = max(n for _, _, n in who)
        floats = 0 if walk else ops.linear_state_workspace_floats(len(sl), longest, H, D, E)
        ws = torch.full((floats,), float("nan"), device=device) if floats else None
        ops.linear_state(src, 0, H * D, 2 * H * D, state, ints(q_start, device), ints(sl, device), 0, len(sl), out, H, D, E, walk=walk,
                         max_q_len=longest, workspace=ws, decay=torch.tensor(decay, device=device), activation="silu")
        for j, (s, lo, n) in enumerate(who):
            outs[s][lo:lo + n] = out[q_start[j]:q_start[j + 1]]
    for s in range(3):
        err = (outs[s].double().cpu() - cases[s][1]).abs().max() / cases[s][1].abs().max()
        assert err < 1e-5, (s, float(err))
    assert torch.equal(state[1], untouched)


def test_lightning_states_in_segments(device):
    """Two portions of 1,003 and 517 tokens of one launch, long enough that each is cut into segments for separate
    workgroups; then a portion that continues from the state they leave."""
    from tessweave_engine_amd.kernels import ops
    H, D, E = 3, 48, 33
    total, first, decay = [1043, 530], [1003, 517], [0.9995, 0.7, 1.0]
    cases = [lightning_rows(H, D, E, T, decay, 7 + T) for T in total]
    assert ops.linear_state_workspace_floats(2, max(first), H, D, E) > 0
    state = torch.zeros(2, H, 48, 48, device=device)
    got = [[], []]
    for lo, hi in (([0, 0], first), (first, total)):
        rows = torch.cat([cases[s][0][lo[s]:hi[s]] for s in range(2)]).to(device)
        starts = [0, hi[0] - lo[0], hi[0] - lo[0] + hi[1] - lo[1]]
        longest = max(hi[s] - lo[s] for s in range(2))
        floats = ops.linear_state_workspace_floats(2, longest, H, D, E)
        ws = torch.full((floats,), float("nan"), device=device) if floats else None
        out = torch.full((rows.shape[0], H * E), float("nan"), device=device)
        ops.linear_state(rows, 0, H * D, 2 * H * D, state, ints(starts, device), ints([1, 0], device), 0, 2, out, H, D, E, walk=False,
                         max_q_len=longest, workspace=ws, decay=torch.tensor(decay, device=device), activation="silu")
        for s in range(2):
            got[s].append(out[starts[s]:starts[s + 1]].double().cpu())
    for s in range(2):
        err = (torch.cat(got[s]) - cases[s][1]).abs().max() / cases[s][1].abs().max()
        assert err < 2e-5, (s, float(err))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("W", [7, 60, 512, 640, 5000])
def test_norm_then_gate(device, dtype, W):
    from tessweave_engine_amd.kernels import ops
    g = torch.Generator().manual_seed(W)
    rows, w = torch.randn(9, 2 * W + 3, generator=g), 1.0 + 0.3 * torch.randn(W, generator=g)
    out = torch.empty(9, W, dtype=tdtype(dtype), device=device)
    dev = rows.to(device)
    ops.gate_group_norm(dev[:, :W], dev[:, W + 3:], w.to(device), out, 1, 1e-5, after=True, scale=0.6)
    want = 0.6 * plain.rms_norm(rows[:, :W].double(), w.double(), 1e-5) * torch.sigmoid(rows[:, W + 3:].double())
    tol = 1e-5 if dtype == "float32" else 1e-2
    assert torch.allclose(out.double().cpu(), want, atol=tol, rtol=tol)


@pytest.mark.parametrize("n", [37, 203, 1001])
@pytest.mark.parametrize("C,X,top,groups", [(72, 70, 4, (7, 3)), (90, 6, 3, (6, 4)), (64, 1, 1, (1, 1)), (2048, 64, 6, (8, 2)), (88, 5, 5, (1, 1)),
                                            (64, 1000, 8, (100, 7)), (64, 1024, 3, (512, 2)), (40, 12, 2, (4, 4)), (64, 16, 3, (2, 1))])
def test_router_with_groups(device, C, X, top, groups, n):
    from tessweave_engine_amd.kernels import ops
    g = torch.Generator().manual_seed(C + X)
    h = torch.randn(n, C, generator=g).to(device)
    router = (2.0 * torch.randn(X, C, generator=g) / math.sqrt(C)).to(device)
    ids = torch.empty(n, top, dtype=torch.int32, device=device)
    weights = torch.empty(n, top, device=device)
    ops.moe_route(h, router, top, ids, weights, groups=groups, scale=1.7)
    s = torch.sigmoid(h.double() @ router.double().T).cpu()
    want, margin = plain.choose_experts(s, {"experts": X, "top": top, "groups": {"count": groups[0], "keep": groups[1]}})
    sure = margin > 1e-5
    assert sure.float().mean() > 0.9
    chosen = ids.long().cpu()
    assert torch.equal(chosen[sure].sort(-1).values, want[sure].sort(-1).values)
    assert torch.allclose(weights.double().cpu(), 1.7 * torch.gather(s, 1, chosen), atol=1e-5)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("n,C,X,top,F", [(1, 88, 5, 2, 40), (9, 128, 16, 4, 64), (300, 96, 3, 3, 24), (130, 72, 64, 1, 100), (17, 64, 1, 1, 32),
                                         (40, 50, 2, 2, 20), (64, 256, 2, 1, 40), (32, 128, 3, 2, 17), (513, 200, 8, 2, 50)])
def test_plain_experts_left_apart_and_summed(device, dtype, n, C, X, top, F):
    """The experts' rows left for a norm to add up, and the same summed (with a shared expert's split-K sums)."""
    from tessweave_engine_amd.kernels import ops
    dt = tdtype(dtype)
    g = torch.Generator().manual_seed(n + X)
    h = torch.randn(n, C, generator=g).to(device).to(dt)
    ups = (torch.randn(X, F, C, generator=g) / math.sqrt(C)).to(dt)
    downs = (torch.randn(X, C, F, generator=g) / math.sqrt(F)).to(dt)
    ids = torch.stack([torch.randperm(X, generator=g)[:top] for _ in range(n)]).to(torch.int32).to(device)
    weights = torch.rand(n, top, generator=g).to(device)
    Cd, Fd = ops.moe_pad(C), ops.moe_pad(F)
    up, down = torch.zeros(X, Fd, Cd, dtype=dt, device=device), torch.zeros(X, C, Fd, dtype=dt, device=device)
    up[:, :F, :C], down[:, :, :F] = ups.to(device), downs.to(device)
    up, down = ops.moe_blocked(up), ops.moe_blocked(down)

    def scratch(tag, shape, dtype_):
        return torch.empty(shape, dtype=dtype_, device=device)
    hd = h.double().cpu()
    each = torch.zeros(n, top, C, dtype=torch.float64)
    for e in range(X):
        y = plain.relu_squared_ff(hd, ups[e].double(), downs[e].double())
        each += (ids.cpu() == e).unsqueeze(-1) * y.unsqueeze(1)
    tol = 2e-5 if dtype == "float32" else 6e-2
    rows, pos = ops.moe_experts(h, ids, weights, None, up, down, 0.0, None, scratch, kind="relu_squared")
    assert torch.allclose(rows.double().cpu()[pos.long().cpu()].view(n, top, C), each, atol=tol, rtol=tol)
    want = (each * weights.double().cpu().unsqueeze(-1)).sum(1)
    more = torch.randn(3, n, C, generator=g)
    x = torch.full((n, C), float("nan"), device=device)
    ops.moe_experts(h, ids, weights, None, up, down, 0.0, x, scratch, kind="relu_squared", accumulate=False, more=more.to(device))
    assert torch.allclose(x.double().cpu(), want + more.double().sum(0), atol=2 * tol, rtol=tol)


# ---------------------------------------------------------------------------------------------------------
# whole models

@pytest.fixture(scope="module", params=list(CONFIGS))
def model(request, tmp_path_factory, device):
    name = request.param
    c = CONFIGS[name]
    weights = make_weights(c, seed=len(name))
    folder = write_folder(tmp_path_factory.mktemp("vulosun_" + name), c, weights)
    g = torch.Generator().manual_seed(50 + len(name))
    tokens = {f"r{i}": torch.randint(0, c["vocab"], (n,), generator=g).tolist() for i, n in enumerate(LENGTHS[name])}
    both = {rid: reference(c, weights, toks) for rid, toks in tokens.items()}
    return dict(name=name, config=c, weights=weights, folder=folder, tokens=tokens, want={k: v[0] for k, v in both.items()},
                margin={k: v[1] for k, v in both.items()})


def check_rows(err, dtype, what="", margin=None):
    """ERR: one relative error per row of ONE sequence (or of several, without margins)."""
    err = np.asarray(err)
    assert np.isfinite(err).all(), what
    if dtype == "bfloat16":
        margin = np.full(len(err), np.inf) if margin is None else np.asarray(margin)
        behind = np.cumsum(margin < CLOSE) > 0                     # rows that may have read what a close call left
        sure, rest = err[~behind], err[behind]
        if len(sure):
            assert sure.max() < 3 * BAR[dtype], (what, int(sure.argmax()), float(sure.max()))
            assert (sure > BAR[dtype]).sum() <= max(1, len(sure) // 5), (what, np.nonzero(sure > BAR[dtype])[0].tolist())
            assert np.median(sure) < BAR[dtype], (what, float(np.median(sure)))
        if len(rest):
            assert np.median(rest) < 5 * BAR[dtype], (what, float(np.median(rest)))
    else:
        allowed = BAR[dtype] + 3.0 * getattr(margin, "float32", 0.0)
        assert (err < allowed).all(), (what, int((err / allowed).argmax()), float(err.max()))


def check_all(model, got, dtype, only=None):
    for rid, want in model["want"].items():
        if only is not None and rid not in only:
            continue
        assert np.isfinite(got[rid]).all()
        check_rows(row_error(got[rid], want), dtype, rid, model["margin"][rid])


SHARED = [differential(4, 2, 12, 20, 0.4, rot(100.0, 4, 3.0), 9, 0.2), differential(4, 2, 12, 20, 0.3, rot(100.0, 4, 3.0), 14, 0.7, kv_from=0)]
PLAIN = attention(2, 1, 16, 16, 0.25, rot(1e3, 8))
FEW_LAYERS = {
    "attention": [attention(6, 2, 24, 40, 0.3, rot(1e3, 12))],
    "attention_one_key_head_values_smaller": [attention(5, 1, 30, 8, 0.2, rot(1e4, 30, 2.0))],
    "differential": [differential(4, 2, 20, 24, 0.3, rot(500.0, 8, 2.0), 11, 0.4)],
    "differential_chunk_of_one": [differential(2, 2, 16, 32, 0.3, rot(500.0, 16), 1, 0.5)],
    "differential_chunk_of_a_page": [differential(3, 1, 8, 50, 0.5, rot(500.0, 2), 4, 0.0)],
    "shared_keys_longer_chunks": SHARED,
    "shared_keys_shorter_chunks": [SHARED[0], differential(4, 2, 12, 20, 0.3, rot(100.0, 4, 3.0), 4, 0.7, kv_from=0)],
    "side_by_side": [parallel(left(4, 2, 24, 40, 0.3, rot(100.0, 10)), right(3, 20, 24, [0.5, 0.99, 1.0]))],
    "side_by_side_one_head": [parallel(left(1, 1, 16, 16, 0.5, rot(100.0, 16)), right(1, 64, 20, [0.9]), 1.0, 1.0)],
    "side_by_side_odd": [parallel(left(3, 1, 30, 7, 0.2, rot(100.0, 2)), right(2, 33, 9, [0.7, 0.01]), -0.5, 2.0)],
    "dense": [dict(PLAIN, mlp=dense(72))],
    "dense_odd": [dict(PLAIN, mlp=dense(50))],
    "experts": [dict(PLAIN, mlp=moe(12, 3, 40, 1.5, (4, 2), 56))],
    "experts_alone": [dict(PLAIN, mlp=moe(7, 2, 20, 0.7))],
    "one_expert": [dict(PLAIN, mlp=moe(1, 1, 24, 1.0, (1, 1), 8))],
}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("kind", list(FEW_LAYERS))
def test_each_mechanism_alone_in_a_small_model(device, tmp_path, kind, dtype):
    """One or two layers, whole and then cut (portions, single tokens, beside another request), on small pages (bfloat16: the
    smallest its fast attention kernels take)."""
    c = config(FEW_LAYERS[kind], width=72, vocab=120)
    weights = make_weights(c, seed=3)
    folder = write_folder(tmp_path, c, weights)
    g = torch.Generator().manual_seed(1)
    tokens = {"a": torch.randint(0, 120, (75,), generator=g).tolist(), "b": torch.randint(0, 120, (19,), generator=g).tolist()}
    want = {k: reference(c, weights, v) for k, v in tokens.items()}
    d = Driver(folder, dtype, pages=60, page_size=4 if dtype == "float32" else 8, max_requests=2)
    whole = d.run([[("a", 75), ("b", 19)]], tokens)
    d.at.clear()
    cut = d.run([[("a", 33)], [("a", 2), ("b", 5)], [("a", 17), ("b", 1)]] + [[("a", 1), ("b", 1)]] * 13 + [[("a", 10)]], tokens)
    for got in (whole, cut):
        for k in tokens:
            check_rows(row_error(got[k], want[k][0]), dtype, (kind, k), want[k][1])
    d.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_whole_prompts(model, dtype):
    d = Driver(model["folder"], dtype, pages=40, page_size=8)
    got = d.run([[(rid, len(toks))] for rid, toks in model["tokens"].items()], model["tokens"])
    check_all(model, got, dtype)
    d.close()


def test_stream_after_every_layer(model):
    """float32: the residual stream after each layer against the plain one's."""
    from tessweave_engine_amd.engine.step import StepEntry
    rid = "r0"
    toks = model["tokens"][rid]
    want = []
    plain.forward(model["config"], double(model["weights"]), toks, layers_out=want)
    d = Driver(model["folder"], "float32", pages=24, page_size=8, graphs=False)
    seq = d.cache.open(rid)
    ctx, ordered, _ = d.stepper.prepare([StepEntry(seq, list(toks), [len(toks) - 1])])
    seen = []
    ctx.segment_end = lambda i: seen.append(ctx.scratch("residual", (ctx.n_tokens, model["config"]["width"]), torch.float32).clone())
    with torch.cuda.stream(d.stepper.stream):
        d.stepper.upload(ctx)
        d.model.forward(ctx)
    d.stepper.synchronize()
    d.stepper.finish(ordered)
    assert len(seen) == len(want)
    for i, (got, ref) in enumerate(zip(seen, want)):
        assert torch.allclose(got.cpu().double(), ref, atol=2e-5 * max(1.0, ref.abs().max().item())), i
    d.close()


@pytest.mark.parametrize("dtype,graphs", [("float32", True), ("float32", False), ("bfloat16", True)])
def test_token_by_token(model, dtype, graphs):
    """Every token decoded alone from the first on (the first tokens of a sequence included)."""
    rid = "r0"
    d = Driver(model["folder"], dtype, pages=24, page_size=4, graphs=graphs)
    got = d.run([[(rid, 1)] for _ in model["tokens"][rid]], {rid: model["tokens"][rid]})
    check_all(model, got, dtype, only=[rid])
    if graphs:
        assert d.model.graph_safe_model and d.stepper.graph_replays > 0
    d.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("sizes", [[2], [3, 1, 2], [16, 5, 2, 2, 9], [7, 8, 1], [10, 17], [64, 48, 2]])
def test_portions(model, dtype, sizes):
    rid = max(model["tokens"], key=lambda r: len(model["tokens"][r]))
    total, schedule, i = len(model["tokens"][rid]), [], 0
    while total:
        n = min(sizes[i % len(sizes)], total)
        schedule.append([(rid, n)])
        total -= n
        i += 1
    d = Driver(model["folder"], dtype, pages=50, page_size=4)
    got = d.run(schedule, {rid: model["tokens"][rid]})
    check_all(model, got, dtype, only=[rid])
    d.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("seed", [0, 1])
def test_unequal_batches_few_pages_two_slots(model, dtype, seed):
    """Portions of some requests beside single tokens of others; at most two requests live, so that every state slot
    is used again, and a page pool that only just holds them."""
    rng = random.Random(seed)
    tokens = model["tokens"]
    pending, live, schedule = list(tokens), {}, []
    while pending or live:
        while pending and len(live) < 2:
            rid = pending.pop(0)
            live[rid] = dict(left=len(tokens[rid]), prompt=rng.randrange(1, len(tokens[rid]) + 1))
        parts = []
        for rid, r in list(live.items()):
            if len(live) > 1 and rng.random() < 0.25:
                continue
            n = min(r["left"], rng.choice([2, 3, 5, 11, 16, 40]) if r["prompt"] > 0 else 1)
            r["prompt"] -= n
            r["left"] -= n
            parts.append((rid, n))
            if r["left"] == 0:
                del live[rid]
        if parts:
            schedule.append(parts)
    page = 8
    longest = sorted(len(t) for t in tokens.values())[-2:]
    pages = sum((n + page - 1) // page for n in longest)
    d = Driver(model["folder"], dtype, pages=pages, page_size=page, max_requests=2)
    got = d.run(schedule, tokens)
    check_all(model, got, dtype)
    d.close()


def test_ways_of_cutting_agree(model):
    """float32: whole, token by token and in portions beside another request differ by rounding only."""
    tokens = model["tokens"]
    rid, other = "r0", "r2"
    runs = []
    for schedule in ([[(rid, len(tokens[rid]))]],
                     [[(rid, 1)] for _ in tokens[rid]],
                     [[(other, 1), (rid, 5)]] + [[(rid, 2), (other, 1)] for _ in range(500)]):
        d = Driver(model["folder"], "float32", pages=50, page_size=4)
        fixed, used = [], {}
        for parts in schedule:
            parts = [(r, min(n, len(tokens[r]) - used.get(r, 0))) for r, n in parts]
            parts = [(r, n) for r, n in parts if n > 0]
            for r, n in parts:
                used[r] = used.get(r, 0) + n
            if parts:
                fixed.append(parts)
        runs.append(d.run(fixed, tokens)[rid])
        d.close()
    for other_run in runs[1:]:
        check_rows(row_error(other_run, runs[0]), "float32", "cuts", model["margin"][rid])


def test_batch_of_many_single_tokens_beside_portions(model):
    """bfloat16 and float32: a step of several single tokens beside two portions gives what each request alone gives."""
    tokens = {k: v for k, v in model["tokens"].items() if len(v) > 6}
    for dtype in ("float32", "bfloat16"):
        d = Driver(model["folder"], dtype, pages=120, page_size=4, max_requests=len(tokens))
        names = list(tokens)
        got = {rid: np.zeros((len(t), model["config"]["vocab"]), dtype=np.float32) for rid, t in tokens.items()}
        parts = [[(rid, 4 + i) if i % 2 else (rid, 1) for i, rid in enumerate(names)],
                 [(rid, 1) if i % 2 else (rid, 3) for i, rid in enumerate(names)]] + [[(rid, 1) for rid in names if len(tokens[rid]) > 8]]
        for p in parts:
            p = [(rid, min(n, len(tokens[rid]) - d.at.get(rid, 0))) for rid, n in p]
            for rid, (lo, rows) in d.step([x for x in p if x[1] > 0], tokens).items():
                got[rid][lo:lo + len(rows)] = rows
        for rid in names:
            n = d.at[rid]
            margin = np.asarray(model["margin"][rid][:n]).view(Slack)
            margin.float32 = model["margin"][rid].float32[:n]
            # (the spread of the whole sequence's logits scales the errors, as everywhere)
            err = row_error(np.concatenate([got[rid][:n], model["want"][rid][n:]]), model["want"][rid])[:n]
            check_rows(err, dtype, rid, margin)
            d.end(rid)
        d.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["odd", "wide"])
def test_far_keys_over_a_long_prompt(device, tmp_path, dtype, name):
    """Query heads that match their own key head's rows: a token's score is by far the largest against the same token
    earlier on, hundreds of tokens back, at page borders, at chunk edges or before a portion's start. 600 tokens of a small
    alphabet: 330 in one step, then portions of 64, 15, 2 and single tokens, on small pages in an order of their own."""
    c = CONFIGS[name]
    weights = make_weights(c, seed=13, sharp=2.0)
    folder = write_folder(tmp_path, c, weights)
    toks = torch.randint(0, 60, (600,), generator=torch.Generator().manual_seed(4)).tolist()
    want, margin = reference(c, weights, toks)
    d = Driver(folder, dtype, pages=180, page_size=4 if dtype == "float32" else 8, max_step_tokens=64)
    warm = {"w0": toks[:37], "w1": toks[:90]}
    d.step([("w0", 36), ("w1", 89)], warm)
    d.end("w0")
    schedule = [[("a", 330)], [("a", 64)], [("a", 15)], [("a", 2)]] + [[("a", 1)]] * 9 + [[("a", 90)], [("a", 90)]]
    got = d.run(schedule, {"a": toks})["a"]
    d.end("w1")
    check_rows(row_error(got, want), dtype, name, margin)
    d.close()


def test_a_chunk_ends_where_it_should(device, tmp_path):
    """A prompt whose first 24 tokens differ (or one of them, the last before a chunk begins) gives the same rows from the
    24th position on, bit for bit where the cut is the same, and other rows before it: nothing of an ended chunk is seen. In
    prompts, in portions cut inside chunks, and decoded."""
    c = config([differential(4, 2, 16, 24, 0.6, rot(100.0, 8), 24, 0.3, mlp=dense(40))], width=64, vocab=50)
    weights = make_weights(c, seed=4, sharp=1.5)
    folder = write_folder(tmp_path, c, weights)
    base = torch.randint(0, 50, (80,), generator=torch.Generator().manual_seed(9)).tolist()
    tokens = {"a": base, "b": [(t + 7) % 50 for t in base[:24]] + base[24:], "c": base[:23] + [(base[23] + 1) % 50] + base[24:]}
    want = {k: reference(c, weights, v)[0] for k, v in tokens.items()}
    assert np.array_equal(want["a"][24:], want["b"][24:]) and row_error(want["a"], want["c"])[23] > 1e-2
    for dtype in ("float32", "bfloat16"):
        for sizes in ([80], [10, 30, 2, 38], [20] + [1] * 60):
            d = Driver(folder, dtype, pages=60, page_size=4, max_requests=3)
            got = {k: d.run([[(k, n)] for n in sizes], {k: tokens[k]})[k] for k in tokens}
            d.close()
            for k in tokens:
                check_rows(row_error(got[k], want[k]), dtype, (k, sizes))
                assert np.array_equal(got["a"][24:], got[k][24:]), (dtype, sizes, k)


def test_a_state_that_remembers_its_first_tokens(device, tmp_path):
    """One layer that forgets nothing: the logits at the end depend on the first tokens. Two prompts that differ in their
    first three tokens only must differ at token 200 and later, and each must match the plain implementation whether it ran
    whole, or in portions and single tokens."""
    c = config([parallel(left(2, 1, 16, 16, 0.2, rot(100.0, 8)), right(2, 64, 48, [1.0, 0.9999]), 1.0, 1.0)], width=64, vocab=50)
    weights = make_weights(c, seed=4)
    weights["l0.mix.left.v"] = weights["l0.mix.left.v"] * 0.0          # (the attention beside it sees them too)
    folder = write_folder(tmp_path, c, weights)
    base = torch.randint(0, 50, (260,), generator=torch.Generator().manual_seed(9)).tolist()
    tokens = {"a": base, "b": [(t + 7) % 50 for t in base[:3]] + base[3:]}
    want = {k: reference(c, weights, v) for k, v in tokens.items()}
    assert row_error(want["a"][0][200:], want["b"][0][200:]).min() > 3e-4
    d = Driver(folder, "float32", pages=40, page_size=16, max_requests=2)
    got = d.run([[("a", 260)], [("b", 100)], [("b", 2)]] + [[("b", 1)]] * 17 + [[("b", 141)]], tokens)
    for k in tokens:
        check_rows(row_error(got[k], want[k][0]), "float32", k, want[k][1])
    d.close()


def random_config(seed):
    """A configuration nobody chose: one to six layers of all kinds in any order, any feed-forward, sizes of every parity,
    differential layers that read earlier ones."""
    rng = random.Random(seed)
    layers = []
    for i in range(rng.randint(1, 6)):
        mlp = None
        kind = rng.random()
        if kind < 0.3:
            mlp = dense(rng.choice([8, 20, 48, 70]))
        elif kind < 0.85:
            experts = rng.choice([1, 2, 6, 9, 32])
            count = rng.choice([n for n in (1, 2, 3, 4, 9) if experts % n == 0])
            keep = rng.randint(1, count)
            mlp = moe(experts, rng.randint(1, min(keep * (experts // count), 4)), rng.choice([8, 20, 48, 70]), rng.uniform(0.3, 2.5),
                      (count, keep) if count > 1 or rng.random() < 0.5 else None, rng.choice([None, 12, 40]))
        G = rng.choice([1, 2, 3])
        H, D, E, scale = G * rng.choice([1, 2, 4]), rng.choice([8, 13, 34, 64, 80]), rng.choice([8, 12, 33, 64, 96]), rng.uniform(0.05, 0.5)
        r = rot(rng.choice([50.0, 1e4, 1e6]), rng.choice([n for n in (2, 4, 12, D // 2 * 2) if n <= D]), rng.choice([None, 1.0, 3.5]))
        pick = rng.random()
        own = [j for j, lay in enumerate(layers) if lay["type"] == "attention_2" and "kv_from" not in lay["mixer"]]
        if pick < 0.3:
            layers.append(attention(H, G, D, E, scale, r, mlp))
        elif pick < 0.5 and own:
            j = rng.choice(own)
            m = layers[j]["mixer"]
            layers.append(differential(m["heads"], m["kv_heads"], m["dim"], m["vdim"], scale, m["rot"], rng.choice([1, 5, 16, 21, 64]), rng.uniform(0, 0.9),
                                       mlp, kv_from=j))
        elif pick < 0.7:
            layers.append(differential(H, G, D, E, scale, r, rng.choice([1, 5, 16, 21, 64, 500]), rng.uniform(0, 0.9), mlp))
        else:
            n = rng.choice([1, 2, 3])
            layers.append(parallel(left(H, G, D, E, scale, r), right(n, rng.choice([4, 9, 16, 50, 96, 130]), rng.choice([3, 8, 20, 64, 100]),
                                                                     [rng.choice([1.0, 0.99, 0.6, 0.1]) for _ in range(n)]),
                                   rng.uniform(-1, 1.5), rng.uniform(-1, 1.5), mlp))
    return config(layers, width=rng.choice([40, 51, 56, 100, 136, 192]), vocab=rng.randint(30, 400), eps=rng.choice([1e-6, 1e-5, 1e-3]))


@pytest.mark.parametrize("seed", list(range(14)))
def test_configurations_drawn_at_random(device, tmp_path, seed):
    """Whole prompts in one batch, then a prompt in portions with its last tokens one by one beside another request, in
    both precisions, for sizes nobody chose."""
    c = random_config(seed)
    weights = make_weights(c, seed=100 + seed)
    folder = write_folder(tmp_path, c, weights)
    g = torch.Generator().manual_seed(seed)
    tokens = {"a": torch.randint(0, c["vocab"], (83,), generator=g).tolist(), "b": torch.randint(0, c["vocab"], (21,), generator=g).tolist()}
    want = {k: reference(c, weights, v) for k, v in tokens.items()}
    for dtype in ("float32", "bfloat16"):
        d = Driver(folder, dtype, pages=40, page_size=4 if seed % 3 == 0 else 16, max_requests=2)
        whole = d.run([[("a", 83), ("b", 21)]], tokens)
        cut = d.run([[("a", 30)], [("a", 17), ("b", 2)], [("a", 2), ("b", 1)], [("a", 24), ("b", 9)]] + [[("a", 1), ("b", 1)]] * 10, tokens)
        for got in (whole, cut):
            for k in tokens:
                check_rows(row_error(got[k], want[k][0]), dtype, (seed, c["width"], k), want[k][1])
        d.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_prompt_in_one_step(device, tmp_path, dtype):
    """1,300 tokens: 1,100 in one step (recurrences over many chunks and segments, prompt attention over many tiles, experts
    with hundreds of rows each), then a portion of 150 behind them and single tokens, beside a second, short request."""
    c = CONFIGS["odd"]
    weights = make_weights(c, seed=17)
    folder = write_folder(tmp_path, c, weights)
    g = torch.Generator().manual_seed(6)
    tokens = {"a": torch.randint(0, c["vocab"], (1300,), generator=g).tolist(), "b": torch.randint(0, c["vocab"], (40,), generator=g).tolist()}
    want = {k: reference(c, weights, v) for k, v in tokens.items()}
    d = Driver(folder, dtype, pages=100, page_size=16, max_requests=2)
    got = d.run([[("a", 1100), ("b", 3)], [("a", 150), ("b", 1)]] + [[("a", 1), ("b", 1)]] * 36 + [[("a", 14)]], tokens)
    for k in tokens:
        check_rows(row_error(got[k], want[k][0]), dtype, k, want[k][1])
    d.close()


def test_long_decoding_from_graphs(device, tmp_path):
    """400 tokens decoded one by one from graphs after a short prompt, two requests side by side."""
    c = CONFIGS["odd"]
    weights = make_weights(c, seed=11)
    folder = write_folder(tmp_path, c, weights)
    g = torch.Generator().manual_seed(3)
    tokens = {"a": torch.randint(0, c["vocab"], (420,), generator=g).tolist(),
              "b": torch.randint(0, c["vocab"], (409,), generator=g).tolist()}
    want = {k: reference(c, weights, v) for k, v in tokens.items()}
    d = Driver(folder, "float32", pages=70, page_size=16)
    got = d.run([[("a", 20), ("b", 9)]] + [[("a", 1), ("b", 1)] for _ in range(400)], tokens)
    for k in tokens:
        check_rows(row_error(got[k], want[k][0]), "float32", k, want[k][1])
    assert d.stepper.graph_replays > 300
    d.close()


@pytest.mark.parametrize("name", ["odd", "wide"])
def test_greedy_generation_through_the_scheduler(device, tmp_path, name):
    """`engine_for(...).generate`: the package's entry point, scheduler, sampler and lookahead. Every generated
    token must be the plain implementation's best token for the text so far (checked where its lead is clear)."""
    from tessweave_engine_amd.cli import engine_for
    c = CONFIGS[name]
    weights = make_weights(c, seed=21)
    folder = write_folder(tmp_path, c, weights)
    g = torch.Generator().manual_seed(8)
    prompts = [torch.randint(0, c["vocab"], (n,), generator=g).tolist() for n in (5, 23, 1, 40, 12, 30)]
    engine = engine_for(folder, dtype="float32", max_context=128, kv_blocks=60, block_size=8, max_active=3,
                        prefill_chunk=16, no_prefix_cache=False)
    try:
        outputs = engine.generate(prompts, max_tokens=24, temperature=0.0)
    finally:
        engine.close()
    clear = 0
    for prompt, out in zip(prompts, outputs):
        assert len(out) == 24
        logits = plain.forward(c, double(weights), prompt + out)[len(prompt) - 1:-1]
        top = logits.topk(2, -1)
        for t, token in enumerate(out):
            if top.values[t, 0] - top.values[t, 1] > 1e-3:
                assert token == int(top.indices[t, 0]), (t, token)
                clear += 1
    assert clear > 100
