"""The Darolix design on the GPU against the plain implementation (`plain_darolix.py`).

Mechanisms alone (each kernel against the plain function of the same mechanism: sinusoidal positions far out, normed
results side by side, the normed and tempered queries with attention behind them made sharp so that one key among hundreds
carries the row, the router with its correction, the grouped experts with identities, the decaying matrix states walked, in
chunks and in segments over cut sequences in reused slots, with decays from one to almost nothing, the decays' logarithms,
the gated norm in parts), then each mixer alone in a model of one layer, then whole models through the package's loader,
cache manager and step function: prefill against token-by-token decoding, portions down to two tokens, unequal batches
against each request alone, few pages and slots that are freed and used again, a long prompt, a state that must survive
hundreds of tokens, long decoding from HIP graphs, sizes drawn at random, and greedy generation through the scheduler.

Bars: float32 rows must agree with the float64 plain implementation to 2e-5 of the logits' spread (the kernels sum in other
orders) plus three times what the PLAIN implementation run in float32 is off by in that row. bfloat16 rows must agree to 3 %
of the spread, one in five up to three times as far (the narrow models here round coarsely). A token whose expert scores
nearly tie between the last expert chosen and the next (`plain.router_margin` under CLOSE) may go the other way in bfloat16,
and what it leaves in the recurrent states and the caches reaches every later row of its sequence: rows behind a sequence's
first such token are only held to a typical error within five times the bar. Every kernel that runs in bfloat16 is the same
template as in float32.
"""
import math
import random

import numpy as np
import pytest
import torch

import plain_darolix as plain
from darolix_util import (CONFIGS, RANKS, Driver, config, left, make_weights, mamba2, moe, parallel, right, row_error,
                          write_folder)

pytestmark = pytest.mark.gpu

BAR = {"float32": 2e-5, "bfloat16": 3e-2}
CLOSE = 0.03         # a margin of scores (they sum to one) under this may go the other way in bfloat16
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
@pytest.mark.parametrize("width", [88, 51, 1, 640])
def test_embedding_with_sinusoids_far_out(device, dtype, width):
    from tessweave_engine_amd.kernels import ops
    g = torch.Generator().manual_seed(width)
    table = torch.randn(30, width, generator=g).to(tdtype(dtype))
    positions = [0, 1, 2, 63, 999, 4097, 30000, 250001]
    toks = [5, 29, 0, 7, 7, 1, 13, 28]
    i = torch.arange((width + 1) // 2, dtype=torch.float64)
    exact = 10000.0 ** (-2.0 * i / width)
    freq = exact.float()
    rest = (exact - freq.double()).float()
    x, copy = torch.empty(8, width, device=device), torch.empty(8, width, device=device)
    feed = ints([28, 1], device)
    ids = ints([5, 29, 0, 7, 7, -2, 13, -1], device)                # the sixth and the last come from the feed
    ops.embed_sinusoid(ids, table.to(device), ints(positions, device), freq.to(device), rest.to(device), 3.7, x, copy=copy, feed=feed)
    want = torch.stack([3.7 * table[t].double() + plain.sinusoids(1, width, torch.float64, start=p)[0] for t, p in zip(toks, positions)])
    assert torch.equal(x, copy)
    assert (x.double().cpu() - want).abs().max() < 2e-6


@pytest.mark.parametrize("n,C,splits", [(5, 88, (1, 3)), (70, 1000, (2, 1)), (3, 4097, (1, 1)), (2, 9000, (2, 2)), (4, 4096, (1,)),
                                        (3, 50, (1, 2, 1, 3))])
def test_normed_results_side_by_side(device, n, C, splits):
    from tessweave_engine_amd.kernels import ops
    g = torch.Generator().manual_seed(n + C)
    x = torch.randn(n, C, generator=g)
    results, want = [], x.double()
    for k, s in enumerate(splits):
        y = torch.randn(s, n, C, generator=g) * 3.0
        w = 1.0 + 0.3 * torch.randn(C, generator=g)
        want = want + (0.5 + k) * plain.rms_norm(y.double().sum(0), w.double(), 1e-5)
        results.append(((y if s > 1 else y[0]).to(device).contiguous(), w.to(device), 0.5 + k))
    got = x.to(device)
    ops.add_normed_sum(got, results, 1e-5)
    assert torch.allclose(got.double().cpu(), want, atol=1e-5 * len(splits))
    before = got.clone()
    ops.add_values(got, before)
    assert torch.equal(got, 2 * before)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("parts,size", [(1, 60), (4, 15), (3, 64), (8, 512), (2, 2500), (5, 1)])
def test_gate_then_norm_in_parts(device, dtype, parts, size):
    from tessweave_engine_amd.kernels import ops
    g = torch.Generator().manual_seed(parts * size)
    n, W = 7, parts * size
    rows = torch.randn(n, 2 * W + 3, generator=g)
    w = 1.0 + 0.3 * torch.randn(W, generator=g)
    out = torch.empty(n, W, dtype=tdtype(dtype), device=device)
    dev = rows.to(device)
    ops.gate_group_norm(dev[:, :W], dev[:, W + 3:], w.to(device), out, parts, 1e-5)
    want = plain.grouped_rms_norm(rows[:, :W].double() * plain.silu(rows[:, W + 3:].double()), w.double(), parts, 1e-5)
    assert torch.allclose(out.double().cpu(), want, atol=1e-5 if dtype == "float32" else 1e-2, rtol=1e-5 if dtype == "float32" else 1e-2)


@pytest.mark.parametrize("n,rank,channels,tau", [(1, 1, 9, 1.0), (19, 16, 300, 16.0), (33, 130, 64, 2.5)])
def test_logarithms_of_the_decays(device, n, rank, channels, tau):
    from tessweave_engine_amd.kernels import ops
    g = torch.Generator().manual_seed(rank)
    low, up = torch.randn(n, rank + 5, generator=g), torch.randn(channels, rank, generator=g)
    bias = 6.0 * torch.randn(channels, generator=g)
    out = torch.empty(n, channels, device=device)
    ops.decay_logs(low.to(device)[:, 2:2 + rank], up.t().contiguous().to(device), bias.to(device), tau, out)
    z = low[:, 2:2 + rank].double() @ up.double().T + bias.double()
    assert torch.allclose(out.double().cpu(), -plain.softplus(-z) / tau, atol=1e-6, rtol=2e-5)


def linear_state_case(H, G, D, E, T, form, seed):
    """Rows [q | k | v] and the decays of one sequence, with the plain result [T, H, E]. form: "head", or the channel form
    with "mild" decays, "mixed" ones (from one to e^-9) or "wild" ones (elements that forget everything at every token)."""
    g = torch.Generator().manual_seed(seed)
    rows = torch.randn(T, 2 * G * D + H * E, generator=g)
    q, k = rows[:, :G * D].double().view(T, G, D), rows[:, G * D:2 * G * D].double().view(T, G, D)
    v = rows[:, 2 * G * D:].double().view(T, H, E)
    out = torch.zeros(T, H, E, dtype=torch.float64)
    if form == "head":
        raw = torch.randn(T, H, generator=g) * 2.0
        dt_bias, A_log, skip = (torch.randn(H, generator=g) for _ in range(3))
        for a in range(H):
            j = a // (H // G)
            dt = plain.softplus(raw[:, a].double() + dt_bias[a].double())
            out[:, a] = plain.state_space_steps(v[:, a], k[:, j], q[:, j] * 0.7, dt, A_log[a].double(), skip[a].double())
        return rows, dict(raw=raw, dt_bias=dt_bias, A_log=A_log, skip=skip), out
    scale = {"mild": 0.1, "mixed": 3.0, "wild": 60.0}[form]
    logs = -scale * torch.rand(T, H * D, generator=g) ** 4
    if form == "wild":
        logs[:, 1::3] *= 1e-3                                       # beside elements that remember
    alpha = torch.exp(logs.double()).view(T, H, D)
    for a in range(H):
        out[:, a] = plain.linear_attention_steps(q[:, a // (H // G)] * 0.7, k[:, a // (H // G)], v[:, a], alpha[:, a])
    return rows, dict(logs=logs), out


@pytest.mark.parametrize("walk", [True, False], ids=["walked", "chunks"])
@pytest.mark.parametrize("form", ["head", "mild", "mixed", "wild"])
@pytest.mark.parametrize("H,G,D,E", [(3, 3, 20, 24), (1, 1, 13, 10), (4, 2, 128, 64), (6, 1, 32, 80), (2, 2, 256, 16), (2, 1, 64, 200),
                                     (4, 4, 100, 7), (8, 2, 12, 70)])
def test_decaying_states_over_cut_sequences_in_reused_slots(device, H, G, D, E, form, walk):
    """Three sequences cut differently (one whole, one in portions of 1, 2, 5 and 33 tokens, one token by token), their
    states in slots that other sequences used before."""
    from tessweave_engine_amd.kernels import ops
    if form != "head" and G != H:
        G = H
    Dp, Ep = (D + 15) // 16 * 16, (E + 15) // 16 * 16
    cuts = [[170], [1, 2, 5, 33, 1, 2, 5, 10], [1] * 23]
    cases = [linear_state_case(H, G, D, E, sum(cut), form, H * D + s) for s, cut in enumerate(cuts)]
    if form == "head":                                              # per-head constants are the layer's, not the sequence's
        for s in (1, 2):
            rows, more, _ = cases[s]
            for key in ("dt_bias", "A_log", "skip"):
                more[key] = cases[0][1][key]
            v = rows[:, 2 * G * D:].double().view(-1, H, E)
            q, k = rows[:, :G * D].double().view(-1, G, D), rows[:, G * D:2 * G * D].double().view(-1, G, D)
            for a in range(H):
                dt = plain.softplus(more["raw"][:, a].double() + more["dt_bias"][a].double())
                cases[s][2][:, a] = plain.state_space_steps(v[:, a], k[:, a // (H // G)], q[:, a // (H // G)] * 0.7, dt,
                                                            more["A_log"][a].double(), more["skip"][a].double())
    state = torch.randn(4, H, Ep, Dp, device=device)
    slots = [2, 0, 3]
    untouched = state[1].clone()
    for s in slots:
        state[s].zero_()
    at = [0, 0, 0]
    outs = [torch.zeros(sum(cut), H * E, device=device) for cut in cuts]
    while any(cuts):
        rows, extra, q_start, sl, who = [], [], [0], [], []
        for s in range(3):
            if cuts[s]:
                n = cuts[s].pop(0)
                lo = at[s]
                rows.append(cases[s][0][lo:lo + n])
                extra.append((cases[s][1]["raw"] if form == "head" else cases[s][1]["logs"])[lo:lo + n])
                q_start.append(q_start[-1] + n)
                sl.append(slots[s])
                who.append((s, lo, n))
                at[s] += n
        src, extra = torch.cat(rows).contiguous().to(device), torch.cat(extra).contiguous().to(device)
        out = torch.full((src.shape[0], H * E), float("nan"), device=device)
        longest = max(n for _, _, n in who)
        options = dict(logs=extra) if form != "head" else dict(raw=extra, **{k: cases[0][1][k].to(device) for k in ("dt_bias", "A_log", "skip")})
        ws = None
        if not walk:
            floats = ops.linear_state_workspace_floats(len(sl), longest, H, D, E)
            ws = torch.full((floats,), float("nan"), device=device) if floats else None
        ops.linear_state(src, 0, G * D, 2 * G * D, state, ints(q_start, device), ints(sl, device), 0, len(sl), out, H, D, E, groups=G,
                         q_scale=0.7, walk=walk, max_q_len=longest, workspace=ws, **options)
        for j, (s, lo, n) in enumerate(who):
            outs[s][lo:lo + n] = out[q_start[j]:q_start[j + 1]]
    for s in range(3):
        want = cases[s][2].reshape(-1, H * E)
        err = (outs[s].double().cpu() - want).abs().max() / want.abs().max()
        assert err < 1e-5, (s, float(err))
    assert torch.equal(state[1], untouched)


@pytest.mark.parametrize("form", ["head", "mild", "wild"])
def test_decaying_states_in_segments(device, form):
    """Two portions of 1,003 and 517 tokens of one launch behind states of their own: long enough that each is cut into
    segments for separate workgroups; then a portion that continues from the state they leave."""
    from tessweave_engine_amd.kernels import ops
    H, D, E = 2, 48, 33
    total = [1043, 530]
    first = [1003, 517]
    cases = [linear_state_case(H, H, D, E, T, form, 7) for T in total]
    # (both sequences have the same constants in the head form: the same seed draws rows of different lengths)
    if form == "head":
        more = cases[1][1]
        for key in ("dt_bias", "A_log", "skip"):
            more[key] = cases[0][1][key]
        rows = cases[1][0].double()
        for a in range(H):
            dt = plain.softplus(more["raw"][:, a].double() + more["dt_bias"][a].double())
            cases[1][2][:, a] = plain.state_space_steps(rows[:, 2 * H * D + a * E:2 * H * D + (a + 1) * E], rows[:, (H + a) * D:(H + a + 1) * D],
                                                        rows[:, a * D:(a + 1) * D] * 0.7, dt, more["A_log"][a].double(), more["skip"][a].double())
    assert ops.linear_state_workspace_floats(2, max(first), H, D, E) > 0
    state = torch.zeros(2, H, 48, 48, device=device)
    got = [[], []]
    for lo, hi in (([0, 0], first), (first, total)):
        rows = torch.cat([cases[s][0][lo[s]:hi[s]] for s in range(2)]).to(device)
        key = "raw" if form == "head" else "logs"
        extra = torch.cat([cases[s][1][key][lo[s]:hi[s]] for s in range(2)]).to(device)
        starts = [0, hi[0] - lo[0], hi[0] - lo[0] + hi[1] - lo[1]]
        longest = max(hi[s] - lo[s] for s in range(2))
        floats = ops.linear_state_workspace_floats(2, longest, H, D, E)
        ws = torch.full((floats,), float("nan"), device=device) if floats else None
        out = torch.full((rows.shape[0], H * E), float("nan"), device=device)
        options = dict(logs=extra) if form != "head" else dict(raw=extra, **{k: cases[0][1][k].to(device) for k in ("dt_bias", "A_log", "skip")})
        ops.linear_state(rows, 0, H * D, 2 * H * D, state, ints(starts, device), ints([1, 0], device), 0, 2, out, H, D, E, q_scale=0.7,
                         walk=False, max_q_len=longest, workspace=ws, **options)
        for s in range(2):
            got[s].append(out[starts[s]:starts[s + 1]].double().cpu())
    for s in range(2):
        want = cases[s][2].reshape(-1, H * E)
        err = (torch.cat(got[s]) - want).abs().max() / want.abs().max()
        assert err < 2e-5, (s, float(err))


@pytest.mark.parametrize("H,D,E,rank,tau", [(3, 20, 24, 1, 1.0), (2, 64, 48, 16, 16.0), (1, 13, 10, 7, 0.3), (2, 128, 33, 130, 8.0), (4, 8, 70, 5, 2.0),
                                            (2, 200, 20, 33, 16.0)])
def test_walked_states_that_form_their_decays(device, H, D, E, rank, tau):
    """Steps of one to four tokens a sequence whose decays are given by their low-rank product."""
    from tessweave_engine_amd.kernels import ops
    g = torch.Generator().manual_seed(D + rank)
    Dp, Ep = (D + 15) // 16 * 16, (E + 15) // 16 * 16
    up, bias = torch.randn(H * D, rank, generator=g) / math.sqrt(rank), 2.0 * torch.randn(H * D, generator=g)
    cuts, at = [[4, 1, 2, 1], [1, 3, 1, 4]], [0, 0]
    rows = [torch.randn(sum(c), 2 * H * D + H * E, generator=g) for c in cuts]
    low = [torch.randn(sum(c), rank + 3, generator=g) for c in cuts]
    want = []
    for s in range(2):
        T = len(rows[s])
        alpha = torch.sigmoid(low[s][:, 3:].double() @ up.double().T + bias.double()) ** (1.0 / tau)
        q, k = rows[s][:, :H * D].double().view(T, H, D) * 0.7, rows[s][:, H * D:2 * H * D].double().view(T, H, D)
        v = rows[s][:, 2 * H * D:].double().view(T, H, E)
        want.append(torch.stack([plain.linear_attention_steps(q[:, a], k[:, a], v[:, a], alpha.view(T, H, D)[:, a]) for a in range(H)], 1))
    state = torch.zeros(3, H, Ep, Dp, device=device)
    for i in range(4):
        n = [c[i] for c in cuts]
        src = torch.cat([rows[s][at[s]:at[s] + n[s]] for s in range(2)]).to(device)
        lo = torch.cat([low[s][at[s]:at[s] + n[s]] for s in range(2)]).to(device)
        out = torch.full((sum(n), H * E), float("nan"), device=device)
        ops.linear_state(src, 0, H * D, 2 * H * D, state, ints([0, n[0], sum(n)], device), ints([2, 0], device), 0, 2, out, H, D, E,
                         q_scale=0.7, walk=True, max_q_len=max(n), low_rank=(lo[:, 3:], up.t().contiguous().to(device), bias.to(device), tau))
        for s in range(2):
            got = out[:n[0]] if s == 0 else out[n[0]:]
            ref = want[s].reshape(-1, H * E)[at[s]:at[s] + n[s]]
            assert (got.double().cpu() - ref).abs().max() < 1e-5 * max(1.0, want[s].abs().max().item()), (i, s)
            at[s] += n[s]
    assert not state[1].any()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("H,G,D,E,cap,page", [(4, 2, 24, 20, 30.0, 4), (8, 8, 32, 64, 0.0, 16), (6, 1, 50, 34, 12.0, 8), (3, 3, 128, 96, 25.0, 16),
                                              (10, 2, 64, 64, 20.0, 16), (2, 2, 15, 7, 15.0, 4)])
def test_normed_heads_with_a_temperature_made_sharp(device, dtype, H, G, D, E, cap, page):
    """Per-head norms, temperature, cache write and the attention kernels, against the plain mechanism. Every query is made
    to point at ONE key with a large score: the first, one at a page's end or start, its neighbour, itself, one far back. A
    key lost or seen wrongly moves its row by the size of a value. Two prompt portions, then single tokens."""
    from tessweave_engine_amd.kernels import ops
    T, eps, temperature = 150, 1e-5, (0.4, 16)
    scale = 24.0 / D
    g = torch.Generator().manual_seed(H * D)
    Dp = (max(D, E) + 15) // 16 * 16
    targets = [min(max([0, i // page * page - 1, i // page * page, i - 1, i, i // 2, i - 97][i % 7], 0), i) for i in range(T)]
    k = torch.randn(T, G * D, generator=g)
    v = torch.randn(T, G * E, generator=g)
    q = torch.stack([k[targets[i]].view(G, D).repeat_interleave(H // G, 0).reshape(-1) for i in range(T)]) * 2.0 + \
        0.05 * torch.randn(T, H * D, generator=g)
    src = torch.cat([q, k, v], 1)
    width = src.shape[1]
    eye = torch.eye(width, dtype=torch.float64)
    w = {"q": eye[:H * D], "k": eye[H * D:(H + G) * D], "v": eye[(H + G) * D:], "o": torch.eye(H * E, dtype=torch.float64)}
    m = {"heads": H, "kv_heads": G, "dim": D, "vdim": E, "scale": scale, "softcap": cap, "q_temp": {"coef": temperature[0], "every": temperature[1]}}
    want = plain.normed_attention(src.double(), w, m, eps)
    q_want = plain.rms_unit(src[:, :H * D].double().view(T, H, D), eps) * plain.query_temperature(T, *temperature).view(T, 1, 1)
    dt = tdtype(dtype)
    blocks = (T + page - 1) // page
    order = list(range(blocks + 3))
    random.Random(3).shuffle(order)
    table = order[:blocks]
    keys = torch.full((blocks + 3, G, page, Dp), 50.0, dtype=dt, device=device)          # what other requests left
    values = torch.full((blocks + 3, G, page, Dp), 50.0, dtype=dt, device=device)
    slots = ints([table[t // page] * page + t % page for t in range(T)], device)
    rows, qd = src.to(device), torch.empty(T, H * Dp, dtype=dt, device=device)
    out = torch.full((T, H * Dp), float("nan"), dtype=dt, device=device)
    bt = ints([table + [-1, -1]], device)
    for lo, hi in [(0, 37), (37, 100)] + [(t, t + 1) for t in range(100, T)]:
        n = hi - lo
        ops.head_finish(rows[lo:hi], 0, H * D, (H + G) * D, ints(list(range(lo, hi)), device), qd[lo:hi], keys, values, slots[lo:hi].contiguous(),
                        H, G, D, E, eps, temperature=temperature)
        starts, lens = ints([0, n], device), ints([hi], device)
        if n > 1:
            ops.attn_prefill(qd[lo:hi], keys, values, bt, starts, lens, 0, 1, n, out[lo:hi], H, G, Dp, scale, softcap=cap)
        else:
            ops.attn_decode(qd[lo:hi], keys, values, bt, starts, lens, 0, 1, out[lo:hi], H, G, Dp, scale, softcap=cap)
    got = out.view(T, H, Dp)[:, :, :E].double().cpu().reshape(T, H * E)
    err = (got - want).abs().amax(1)
    tol = 1e-4 if dtype == "float32" else 0.15
    assert err.max() < tol, (int(err.argmax()), targets[int(err.argmax())], float(err.max()))
    q_got = qd.view(T, H, Dp).double().cpu()
    assert torch.allclose(q_got[:, :, :D], q_want, rtol=2e-6 if dtype == "float32" else 5e-3, atol=1e-6) and not q_got[:, :, D:].any()


@pytest.mark.parametrize("n", [37, 203, 1001])
@pytest.mark.parametrize("C,X,top", [(72, 70, 4), (90, 7, 3), (64, 1, 1), (2048, 24, 2), (88, 5, 5)])
def test_router_with_a_correction(device, C, X, top, n):
    from tessweave_engine_amd.kernels import ops
    g = torch.Generator().manual_seed(C + X)
    h = torch.randn(n, C, generator=g).to(device)
    router = (2.0 * torch.randn(X, C, generator=g) / math.sqrt(C)).to(device)
    correction = (0.3 * torch.randn(X, generator=g)).to(device)
    if X > 2:
        router[2] = router[1]
        correction[2] = correction[1]                           # a tie: the lower index wins
    ids = torch.empty(n, top, dtype=torch.int32, device=device)
    weights = torch.empty(n, top, device=device)
    ops.moe_route(h, router, top, ids, weights, bias=correction, weighting="softmax_all")
    s = torch.softmax(h.double() @ router.double().T, -1)
    choice = s + correction.double()
    best = torch.topk(choice, top, dim=-1).values
    assert torch.allclose(torch.gather(choice, 1, ids.long()), best, atol=1e-6)
    mine = torch.gather(s, 1, ids.long())
    assert torch.allclose(weights.double(), mine / mine.sum(-1, keepdim=True), atol=1e-5)
    if X > 2:
        chosen = ids.long()
        both = (chosen == 1).any(-1) ^ (chosen == 2).any(-1)
        assert not (chosen[both] == 2).any()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("n,C,X,identity,top,F", [(1, 88, 5, 2, 2, 40), (9, 128, 16, 0, 4, 64), (300, 96, 3, 3, 3, 24), (130, 72, 64, 8, 1, 100),
                                                  (17, 64, 1, 5, 2, 32), (40, 50, 2, 1, 3, 20), (40, 64, 1, 0, 1, 48),
                                                  (64, 256, 2, 1, 1, 40), (32, 128, 3, 1, 2, 17), (5, 64, 1, 9, 2, 24)])
def test_grouped_experts_with_identities(device, dtype, n, C, X, identity, top, F):
    """Gated experts beside ones that return the input; a mixer's split-K sums go into the same result."""
    from tessweave_engine_amd.kernels import ops
    dt = tdtype(dtype)
    g = torch.Generator().manual_seed(n + X)
    h = torch.randn(n, C, generator=g).to(device).to(dt)
    gates, ups = ((torch.randn(X, F, C, generator=g) / math.sqrt(C)).to(dt) for _ in range(2))
    downs = (torch.randn(X, C, F, generator=g) / math.sqrt(F)).to(dt)
    ids = torch.stack([torch.randperm(X + identity, generator=g)[:top] for _ in range(n)]).to(torch.int32).to(device)
    weights = torch.softmax(torch.randn(n, top, generator=g), -1).to(device)
    Cd, Fd = ops.moe_pad(C), ops.moe_pad(F)
    gate, up = (torch.zeros(X, Fd, Cd, dtype=dt, device=device) for _ in range(2))
    down = torch.zeros(X, C, Fd, dtype=dt, device=device)
    gate[:, :F, :C], up[:, :F, :C], down[:, :, :F] = gates.to(device), ups.to(device), downs.to(device)

    def scratch(tag, shape, dtype_):
        return torch.empty(shape, dtype=dtype_, device=device)
    more = torch.randn(3, n, C, generator=g)
    want = more.double().sum(0)
    hd = h.double().cpu()
    for t in range(n):
        for r in range(top):
            e = int(ids[t, r])
            y = plain.expert(hd[t:t + 1], gates[e].double(), ups[e].double(), downs[e].double())[0] if e < X else hd[t]
            want[t] += weights[t, r].double().cpu() * y
    x = torch.randn(n, C, generator=g).to(device)
    base = x.double().cpu()
    ops.moe_experts(h, ids, weights, ops.moe_blocked(gate), ops.moe_blocked(up), ops.moe_blocked(down), 0.0, x, scratch, kind="silu",
                    more=more.to(device))
    assert torch.allclose(x.double().cpu() - base, want, atol=2e-5 if dtype == "float32" else 4e-2)


# ---------------------------------------------------------------------------------------------------------
# whole models

@pytest.fixture(scope="module", params=list(CONFIGS))
def model(request, tmp_path_factory, device):
    name = request.param
    c = CONFIGS[name]
    weights = make_weights(c, seed=len(name), rank=RANKS[name])
    folder = write_folder(tmp_path_factory.mktemp("darolix_" + name), c, weights)
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


ONE_LAYER = {
    "state_space": mamba2(6, 20, 24, 3, 4, 2),
    "state_space_one_tap_one_head": mamba2(1, 30, 9, 1, 1, 3),
    "state_space_large": mamba2(2, 72, 200, 2, 3, 1),
    "side_by_side": parallel(left(4, 2, 24, 40, 0.3, 10.0, 0.5, 10), right(3, 20, 24, 8.0)),
    "side_by_side_plain": parallel(left(2, 2, 16, 16, 0.5), right(2, 64, 20, 16.0)),
    "side_by_side_fast_decays": parallel(left(3, 1, 30, 8, 0.2, 5.0, -0.1, 3), right(2, 40, 24, 0.05)),
    "experts": mamba2(2, 16, 16, 1, 2, 1, mlp=moe(7, 3, 3, 40)),
    "identities_alone_are_enough": mamba2(2, 16, 16, 1, 2, 1, mlp=moe(1, 6, 2, 24)),
}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("kind", list(ONE_LAYER))
def test_each_mechanism_alone_in_a_model_of_one_layer(device, tmp_path, kind, dtype):
    """One layer that runs twice, whole and then cut (portions, single tokens, beside another request), pages of four
    tokens."""
    c = config([ONE_LAYER[kind]], width=72, vocab=120, scale=5.0, loop=(0, 1, 2))
    weights = make_weights(c, seed=3, rank=7)
    folder = write_folder(tmp_path, c, weights)
    g = torch.Generator().manual_seed(1)
    tokens = {"a": torch.randint(0, 120, (75,), generator=g).tolist(), "b": torch.randint(0, 120, (19,), generator=g).tolist()}
    want = {k: reference(c, weights, v) for k, v in tokens.items()}
    d = Driver(folder, dtype, pages=60, page_size=4, max_requests=2)
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
    """float32: the residual stream after each layer run (repeated ones included) against the plain one's."""
    from tessweave_engine_amd.engine.step import StepEntry
    rid = "r0"
    toks = model["tokens"][rid]
    want = []
    plain.forward(model["config"], double(model["weights"]), toks, layers_out=want)
    d = Driver(model["folder"], "float32", pages=24, page_size=8, graphs=False)
    d.model.defer_sums = False                                  # (a sublayer's sums then are in the stream when its layer ends)
    d.stepper._defer_sums = False
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
@pytest.mark.parametrize("sizes", [[2], [3, 1, 2], [16, 5, 2, 2, 9], [7, 8, 1], [17, 32], [64, 48, 2]])
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
    is used again (recurrent states, convolution inputs), and a page pool that only just holds them."""
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
            margin = model["margin"][rid][:n]
            if hasattr(model["margin"][rid], "float32"):
                margin = np.asarray(margin).view(Slack)
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
    earlier on, hundreds of tokens back, at page borders or before a portion's start. 600 tokens of a small alphabet: 330 in
    one step, then portions of 64, 15, 2 and single tokens, on pages of four tokens in an order of their own."""
    c = dict(CONFIGS[name], embedding={"scale": 30.0})
    weights = make_weights(c, seed=13, rank=RANKS[name], sharp=2.0)
    folder = write_folder(tmp_path, c, weights)
    toks = torch.randint(0, c["vocab"], (600,), generator=torch.Generator().manual_seed(4)).tolist()
    want, margin = reference(c, weights, toks)
    d = Driver(folder, dtype, pages=180, page_size=4, max_step_tokens=64)
    warm = {"w0": toks[:37], "w1": toks[:90]}
    d.step([("w0", 36), ("w1", 89)], warm)
    d.end("w0")
    schedule = [[("a", 330)], [("a", 64)], [("a", 15)], [("a", 2)]] + [[("a", 1)]] * 9 + [[("a", 90)], [("a", 90)]]
    got = d.run(schedule, {"a": toks})["a"]
    d.end("w1")
    check_rows(row_error(got, want), dtype, name, margin)
    d.close()


@pytest.mark.parametrize("kind", ["state_space", "linear_attention"])
def test_a_state_that_remembers_its_first_tokens(device, tmp_path, kind):
    """One layer that forgets nothing: the logits at the end depend on the first tokens. Two prompts that differ in their
    first three tokens only must differ at token 200 and later, and each must match the plain implementation whether it ran
    whole, or in portions and single tokens."""
    layer = mamba2(2, 24, 64, 1, 3, 1) if kind == "state_space" else parallel(left(2, 1, 16, 16, 0.2), right(2, 64, 48, 16.0))
    c = config([layer], width=64, vocab=50, scale=3.0)
    weights = make_weights(c, seed=4)
    if kind == "state_space":
        weights["l0.mix.A_log"] = torch.full((2,), -9.0).to(torch.bfloat16)
    else:
        weights["l0.mix.right.a2.b"] = torch.full((128,), 12.0).to(torch.bfloat16)
        weights["l0.mix.left.v"] = weights["l0.mix.left.v"] * 0.0          # (the attention beside it sees them too)
    folder = write_folder(tmp_path, c, weights)
    g = torch.Generator().manual_seed(9)
    base = torch.randint(0, 50, (260,), generator=g).tolist()
    other = [(t + 7) % 50 for t in base[:3]] + base[3:]
    tokens = {"a": base, "b": other}
    want = {k: reference(c, weights, v) for k, v in tokens.items()}
    assert row_error(want["a"][0][200:], want["b"][0][200:]).min() > 1e-3
    d = Driver(folder, "float32", pages=40, page_size=16, max_requests=2)
    got = d.run([[("a", 260)], [("b", 100)], [("b", 2)]] + [[("b", 1)]] * 17 + [[("b", 141)]], tokens)
    for k in tokens:
        check_rows(row_error(got[k], want[k][0]), "float32", k, want[k][1])
    d.close()


def random_config(seed):
    """A configuration nobody chose: one to five layers of both kinds in any order, any feed-forward, sizes of every
    parity, a loop over any of them."""
    rng = random.Random(seed)
    layers = []
    for _ in range(rng.randint(1, 5)):
        mlp = None
        if rng.random() < 0.75:
            experts, identity = rng.choice([1, 2, 6, 9, 33]), rng.choice([0, 1, 4, 7])
            mlp = moe(experts, identity, rng.randint(1, min(experts + identity, 4)), rng.choice([8, 20, 48, 70]))
        if rng.random() < 0.5:
            G = rng.choice([1, 2, 3])
            H, E = G * rng.choice([1, 2, 4]), rng.choice([6, 16, 20, 48, 66])
            norm = rng.choice([p for p in (1, 2, 3, 4, 6) if (H * E) % p == 0])
            layers.append(mamba2(H, E, rng.choice([4, 9, 16, 50, 96, 130]), G, rng.randint(1, 5), norm, mlp))
        else:
            G = rng.choice([1, 2, 3])
            cap, temp = rng.choice([None, 5.0, 30.0]), rng.choice([(None, None), (0.3, 1), (0.5, 20), (-0.1, 7)])
            layers.append(parallel(left(G * rng.choice([1, 2, 4]), G, rng.choice([8, 13, 34, 64, 80]), rng.choice([8, 12, 33, 64, 96]),
                                        rng.uniform(0.05, 0.5), cap, *temp),
                                   right(rng.choice([1, 2, 3]), rng.choice([4, 9, 16, 50, 96, 130]), rng.choice([3, 8, 20, 64, 100]),
                                         rng.choice([1.0, 4.0, 16.0])), mlp))
    start = rng.randint(0, len(layers) - 1)
    loop = (start, rng.randint(start, len(layers)), rng.randint(1, 3)) if rng.random() < 0.7 else None
    return config(layers, width=rng.choice([40, 56, 100, 136, 192]), vocab=rng.randint(30, 400), scale=rng.choice([1.0, 6.0, 14.1]),
                  loop=loop, eps=rng.choice([1e-6, 1e-5, 1e-3]))


@pytest.mark.parametrize("seed", list(range(12)))
def test_configurations_drawn_at_random(device, tmp_path, seed):
    """Whole prompts in one batch, then a prompt in portions with its last tokens one by one beside another request, in
    both precisions, for sizes nobody chose."""
    c = random_config(seed)
    weights = make_weights(c, seed=100 + seed, rank=1 + 5 * seed)
    folder = write_folder(tmp_path, c, weights)
    g = torch.Generator().manual_seed(seed)
    tokens = {"a": torch.randint(0, c["vocab"], (83,), generator=g).tolist(), "b": torch.randint(0, c["vocab"], (21,), generator=g).tolist()}
    want = {k: reference(c, weights, v) for k, v in tokens.items()}
    for dtype in ("float32", "bfloat16"):
        d = Driver(folder, dtype, pages=40, page_size=4, max_requests=2)
        whole = d.run([[("a", 83), ("b", 21)]], tokens)
        cut = d.run([[("a", 30)], [("a", 17), ("b", 2)], [("a", 2), ("b", 1)], [("a", 24), ("b", 9)]] + [[("a", 1), ("b", 1)]] * 10, tokens)
        for got in (whole, cut):
            for k in tokens:
                check_rows(row_error(got[k], want[k][0]), dtype, (seed, c["width"], k), want[k][1])
        d.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_prompt_in_one_step(device, tmp_path, dtype):
    """1,300 tokens: 1,100 in one step (the recurrences over many chunks and segments, prompt attention over many tiles,
    experts with hundreds of rows each), then a portion of 150 behind them and single tokens, beside a second, short request."""
    c = CONFIGS["odd"]
    weights = make_weights(c, seed=17, rank=RANKS["odd"])
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
    weights = make_weights(c, seed=11, rank=RANKS["odd"])
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
    weights = make_weights(c, seed=21, rank=RANKS[name])
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
