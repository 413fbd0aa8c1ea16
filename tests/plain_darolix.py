"""A plain, slow implementation of the Darolix decoder, one function per mechanism.

Written from the design's equations with ordinary tensor operations on whole sequences; it shares no
code with the package and keeps no cache: a sequence is always computed from its first token. The
tests compare the engine with it (prefill, decoding, portions and batches all have to give what this
gives for the whole sequence).

Notation: T tokens, C the model's width, H heads, G key heads or groups, D the query/key size of a head,
E its value size, N the size of a state-space group's B and C, V the vocabulary, F an expert's inner size.
"""
from __future__ import annotations

import math

import torch


def rms_unit(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def rms_norm(x, w, eps):
    return rms_unit(x, eps) * w


def silu(z):
    return z * torch.sigmoid(z)


def softplus(z):
    return torch.clamp(z, min=0) + torch.log1p(torch.exp(-z.abs()))


def sinusoids(T, width, dtype, start=0):
    """[T, width]: entry 2i of position p is sin(p 10000^(-2i / width)), entry 2i + 1 its cosine. (The angles are formed
    in float64 and rounded with their sines.)"""
    p = torch.arange(start, start + T, dtype=torch.float64).view(-1, 1)
    entry = torch.arange(width)
    angle = p * 10000.0 ** (-2.0 * (entry // 2).to(torch.float64) / width)
    return torch.where(entry % 2 == 0, torch.sin(angle), torch.cos(angle)).to(dtype)


def embed(tokens, table, scale):
    rows = table[torch.as_tensor(tokens, dtype=torch.long)] * scale
    return rows + sinusoids(rows.shape[0], rows.shape[1], rows.dtype)


def causal_taps(u, w):
    """u [T, channels], w [channels, taps]: y_t = sum_j w[:, j] u_(t - taps + 1 + j), zeros before the start."""
    T, taps = u.shape[0], w.shape[1]
    padded = torch.cat([u.new_zeros(taps - 1, u.shape[1]), u], 0)
    y = torch.zeros_like(u)
    for j in range(taps):
        y = y + padded[j:j + T] * w[:, j]
    return y


def state_space_steps(x, B, C, dt, log_rate, D):
    """The state-space recurrence of one head, token by token. x [T, E], B, C [T, N], dt [T]; the state S [N, E] starts
    at zero and decays by exp(-exp(log_rate) dt)."""
    S = x.new_zeros(B.shape[1], x.shape[1])
    out = []
    for t in range(x.shape[0]):
        S = torch.exp(-torch.exp(log_rate) * dt[t]) * S + dt[t] * torch.outer(B[t], x[t])
        out.append(S.T @ C[t] + D * x[t])
    return torch.stack(out)


def grouped_rms_norm(y, w, parts, eps):
    """The row in `parts` equal parts, each divided by its own root mean square; then the weight."""
    T, inner = y.shape
    return rms_unit(y.view(T, parts, inner // parts), eps).reshape(T, inner) * w


def mamba2(h, w, m, eps):
    T = h.shape[0]
    H, E, N, G = m["heads"], m["vdim"], m["state"], m["groups"]
    inner = H * E
    z, xbc, dt = torch.split(h @ w["in"].T, [inner, inner + 2 * G * N, H], -1)
    xbc = silu(causal_taps(xbc, w["conv"]) + w["conv.b"])
    x, B, C = torch.split(xbc, [inner, G * N, G * N], -1)
    x, B, C = x.view(T, H, E), B.view(T, G, N), C.view(T, G, N)
    dt = softplus(dt + w["dt_bias"])
    y = torch.zeros(T, H, E, dtype=h.dtype)
    for a in range(H):
        g = a // (H // G)
        y[:, a] = state_space_steps(x[:, a], B[:, g], C[:, g], dt[:, a], w["A_log"][a], w["D"][a])
    y = y.reshape(T, inner) * silu(z)
    return grouped_rms_norm(y, w["norm"], m["norm_groups"], eps) @ w["o"].T


def query_temperature(T, coef, every):
    """1 + coef ln(floor((p + 1) / every) + 1) for positions p = 0 .. T - 1."""
    return torch.tensor([1.0 + coef * math.log((p + 1) // every + 1) for p in range(T)], dtype=torch.float64)


def normed_attention(h, w, m, eps):
    """Causal attention without rotation whose queries and keys are divided by their root mean square per head, whose
    queries grow with the position, and whose scores pass a soft cap."""
    T = h.shape[0]
    H, G, D, E = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rms_unit((h @ w["q"].T).view(T, H, D), eps)
    k = rms_unit((h @ w["k"].T).view(T, G, D), eps)
    v = (h @ w["v"].T).view(T, G, E)
    if m.get("q_temp"):
        q = q * query_temperature(T, m["q_temp"]["coef"], m["q_temp"]["every"]).to(h.dtype).view(T, 1, 1)
    visible = torch.tril(torch.ones(T, T, dtype=torch.bool))
    out = torch.zeros(T, H, E, dtype=h.dtype)
    for a in range(H):
        g = a // (H // G)
        s = (q[:, a] @ k[:, g].T) * m["scale"]
        if m.get("softcap"):
            s = m["softcap"] * torch.tanh(s / m["softcap"])
        out[:, a] = torch.softmax(s.masked_fill(~visible, -math.inf), -1) @ v[:, g]
    return out.reshape(T, H * E) @ w["o"].T


def linear_attention_steps(q, k, v, alpha):
    """Gated linear attention of one head, token by token. q, k, alpha [T, D], v [T, E]; the state S [D, E] starts at
    zero and its rows decay by alpha."""
    S = q.new_zeros(q.shape[1], v.shape[1])
    out = []
    for t in range(q.shape[0]):
        S = alpha[t].view(-1, 1) * S + torch.outer(k[t], v[t])
        out.append(S.T @ q[t])
    return torch.stack(out)


def gated_linear_attention(h, w, m, eps):
    T = h.shape[0]
    H, D, E = m["heads"], m["dim"], m["vdim"]
    q = (h @ w["q"].T).view(T, H, D) * D ** -0.5
    k = (h @ w["k"].T).view(T, H, D)
    v = (h @ w["v"].T).view(T, H, E)
    z = (h @ w["a1"].T) @ w["a2"].T + w["a2.b"]
    alpha = torch.exp(-softplus(-z) / m["tau"]).view(T, H, D)          # sigmoid(z)^(1 / tau)
    o = torch.stack([linear_attention_steps(q[:, a], k[:, a], v[:, a], alpha[:, a]) for a in range(H)], 1)
    o = rms_norm(o, w["norm"], eps).reshape(T, H * E)
    return (o * silu(h @ w["g"].T)) @ w["o"].T


def side_by_side(h, w, m, eps):
    """Half the sum of two mixers' results, each normed over the model's width."""
    left = normed_attention(h, sub(w, "left."), m["left"], eps)
    right = gated_linear_attention(h, sub(w, "right."), m["right"], eps)
    return 0.5 * (rms_norm(left, w["left.out"], eps) + rms_norm(right, w["right.out"], eps))


def expert(h, gate, up, down):
    return (silu(h @ gate.T) * (h @ up.T)) @ down.T


def router_margin(s, top):
    """Per token, how far the last chosen score lies above the best one left out (infinite if all are chosen)."""
    if top >= s.shape[-1]:
        return torch.full(s.shape[:-1], math.inf, dtype=s.dtype)
    best = torch.topk(s, top + 1, dim=-1).values
    return best[..., top - 1] - best[..., top]


def routed_ff(h, w, mlp, margins=None):
    """A softmax over all experts scores them, a correction decides with it who is chosen, the chosen ones' own scores
    (made to sum to one) weigh their results; the last experts are the identity."""
    top, n = mlp["router"]["top"], mlp["router"]["experts"]
    s = torch.softmax(h @ w["router"].T, -1)
    choice = s + w["correction"]
    if margins is not None:
        margins.append(router_margin(choice, top))
    ids = torch.topk(choice, top, dim=-1).indices
    chosen = torch.zeros_like(s).scatter(-1, ids, 1.0) * s
    share = chosen / (chosen.sum(-1, keepdim=True) + 1e-20)
    out = torch.zeros_like(h)
    for e in range(s.shape[-1]):
        rows = torch.nonzero((ids == e).any(-1)).flatten()
        if len(rows):
            y = expert(h[rows], w[f"e{e}.gate"], w[f"e{e}.up"], w[f"e{e}.down"]) if e < n else h[rows]
            out[rows] = out[rows] + share[rows, e, None] * y
    return out


MIXERS = {"mamba2": mamba2, "parallel": side_by_side}


def sub(weights, prefix):
    """The tensors whose names start with `prefix`, by the rest of their names."""
    return {k[len(prefix):]: v for k, v in weights.items() if k.startswith(prefix)}


def layer_runs(config):
    """[(layer, does a pass but the first begin here)] in the order the layers run."""
    n = len(config["layers"])
    loop = config.get("loop") or {"start": 0, "stop": 0, "times": 1}
    runs = [(i, False) for i in range(loop["start"])]
    for turn in range(loop["times"]):
        runs += [(i, turn > 0 and i == loop["start"]) for i in range(loop["start"], loop["stop"])]
    return runs + [(i, False) for i in range(loop["stop"], n)]


def forward(config, weights, tokens, dtype=torch.float64, layers_out=None, margins=None):
    """Logits [T, V] of a whole sequence. weights: name -> tensor (any float type). layers_out: a list that gets the
    stream after every layer run; margins: a list that gets every routed layer's `router_margin` per token."""
    w = {k: (v.to(dtype) if v.is_floating_point() else v) for k, v in weights.items()}
    eps = config["norm"]["eps"]
    first = x = embed(tokens, w["embed"], config["embedding"]["scale"])
    for i, again in layer_runs(config):
        layer, p = config["layers"][i], f"l{i}."
        if again:
            x = x + first
        h = rms_norm(x, w[p + "norm1"], eps)
        y = MIXERS[layer["type"]](h, sub(w, p + "mix."), layer["mixer"], eps)
        if layer.get("mlp") is not None:
            y = y + routed_ff(h, sub(w, p + "mlp."), layer["mlp"], margins)
        x = x + y
        if layers_out is not None:
            layers_out.append(x.clone())
    return rms_norm(x, w["final.norm"], eps) @ w["head"].T
