"""A plain, slow implementation of the Vulosun decoder, one function per mechanism.

Written from the design's equations with ordinary tensor operations on whole sequences; it shares no
code with the package and keeps no cache: a sequence is always computed from its first token. The
tests compare the engine with it (prefill, decoding, portions and batches all have to give what this
gives for the whole sequence).

Notation: T tokens, C the model's width, H heads, G key heads, D the query/key size of a head, E its
value size, V the vocabulary, F an inner size, X experts.
"""
from __future__ import annotations

import math

import torch


def layer_norm(x, w, b, eps):
    centred = x - x.mean(-1, keepdim=True)
    return centred / torch.sqrt((centred * centred).mean(-1, keepdim=True) + eps) * w + b


def rms_unit(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def rms_norm(x, w, eps):
    return rms_unit(x, eps) * w


def silu(z):
    return z * torch.sigmoid(z)


def angles(T, rot, dtype):
    """[T, dims / 2]: position times base^(-2i / dims), over the scaling's factor if there is one. (Formed in float64.)"""
    i = torch.arange(rot["dims"] // 2, dtype=torch.float64)
    f = rot["base"] ** (-2.0 * i / rot["dims"])
    if rot.get("scaling"):
        f = f / rot["scaling"]["factor"]
    return torch.arange(T, dtype=torch.float64).view(-1, 1) * f


def turn(u, v, a):
    c, s = torch.cos(a).to(u.dtype), torch.sin(a).to(u.dtype)
    return u * c - v * s, v * c + u * s


def rotate_halves(x, rot):
    """x [T, heads, D]: of the first `dims` elements of a head, i turns with i + dims / 2."""
    half = rot["dims"] // 2
    a = angles(x.shape[0], rot, x.dtype).unsqueeze(1)
    u, v = turn(x[..., :half], x[..., half:2 * half], a)
    return torch.cat([u, v, x[..., 2 * half:]], -1)


def rotate_neighbours(x, rot):
    """x [T, heads, D]: of the first `dims` elements of a head, 2i turns with 2i + 1."""
    n = rot["dims"]
    a = angles(x.shape[0], rot, x.dtype).unsqueeze(1)
    u, v = turn(x[..., 0:n:2], x[..., 1:n:2], a)
    return torch.cat([torch.stack([u, v], -1).flatten(-2), x[..., n:]], -1)


def causal(T):
    return torch.tril(torch.ones(T, T, dtype=torch.bool))


def same_chunk(T, size):
    c = torch.arange(T) // size
    return causal(T) & (c.view(-1, 1) == c.view(1, -1))


def attend(q, k, v, scale, visible, sink=None):
    """q [T, H, D], k [T, G, D], v [T, G, E] -> [T, H, E]; sink [H] or None: exp(sink_h) more in the denominator."""
    T, H, G = q.shape[0], q.shape[1], k.shape[1]
    out = []
    for a in range(H):
        g = a // (H // G)
        s = ((q[:, a] @ k[:, g].T) * scale).masked_fill(~visible, -math.inf)
        if sink is not None:
            s = torch.cat([s, sink[a].expand(T, 1)], 1)
        p = torch.softmax(s, -1)[:, :T]
        out.append(p @ v[:, g])
    return torch.stack(out, 1)


def whole_normed_attention(h, w, m, eps):
    """Queries and keys normed over all heads at once, neighbours rotated, a gate per head on the result."""
    T, H, G, D, E = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rms_norm(h @ w["q"].T, w["q.norm"], eps).view(T, H, D)
    k = rms_norm(h @ w["k"].T, w["k.norm"], eps).view(T, G, D)
    v = (h @ w["v"].T).view(T, G, E)
    o = attend(rotate_neighbours(q, m["rot"]), rotate_neighbours(k, m["rot"]), v, m["scale"], causal(T))
    return (o * torch.sigmoid(h @ w["g"].T).unsqueeze(-1)).reshape(T, H * E) @ w["o"].T


def head_normed_attention(h, w, m, eps):
    """Queries and keys normed head by head with one weight for all heads, halves rotated, a sink per head."""
    T, H, G, D, E = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rms_norm((h @ w["q"].T).view(T, H, D), w["q.norm"], eps)
    k = rms_norm((h @ w["k"].T).view(T, G, D), w["k.norm"], eps)
    v = (h @ w["v"].T).view(T, G, E)
    o = attend(rotate_halves(q, m["rot"]), rotate_halves(k, m["rot"]), v, m["scale"], causal(T), w["sink"])
    return o.reshape(T, H * E) @ w["o"].T


def differential_lambda(w, diff):
    return torch.exp((w["lq1"] * w["lk1"]).sum()) - torch.exp((w["lq2"] * w["lk2"]).sum()) + diff


def combine_maps(a1, a2, lam, diff, eps):
    """The two maps' results of a head: their weighted difference over its root mean square, times 1 - diff."""
    return rms_unit(a1 - lam * a2, eps) * (1.0 - diff)


def chunked_keys_values(h, w, m):
    """The keys (both maps, rotated) and values of a differential layer: what a later layer may take over."""
    T, G, D, E = h.shape[0], m["kv_heads"], m["dim"], m["vdim"]
    k = rotate_neighbours((h @ w["k"].T + w["k.b"]).view(T, G * 2, D), m["rot"]).view(T, G, 2, D)
    return k, (h @ w["v"].T + w["v.b"]).view(T, G, E)


def differential_attention(h, w, m, eps, kv=None):
    T, H, D, E = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q = rotate_neighbours((h @ w["q"].T + w["q.b"]).view(T, H * 2, D), m["rot"]).view(T, H, 2, D)
    k, v = kv if kv is not None else chunked_keys_values(h, w, m)
    visible = same_chunk(T, m["mask"]["size"])
    a1, a2 = (attend(q[:, :, i], k[:, :, i], v, m["scale"], visible) for i in (0, 1))
    o = combine_maps(a1, a2, differential_lambda(w, m["diff"]), m["diff"], eps)
    return (o * torch.sigmoid(h @ w["g"].T).unsqueeze(-1)).reshape(T, H * E) @ w["o"].T


def lightning_steps(q, k, v, decay):
    """Linear attention of one head with a fixed decay, token by token. q, k [T, D], v [T, E]; the state [D, E] starts at zero."""
    S = q.new_zeros(q.shape[1], v.shape[1])
    out = []
    for t in range(q.shape[0]):
        S = decay * S + torch.outer(k[t], v[t])
        out.append(S.T @ q[t])
    return torch.stack(out)


def lightning_attention(h, w, m, eps):
    T, H, D, E = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q, k, v = silu(h @ w["q"].T).view(T, H, D), silu(h @ w["k"].T).view(T, H, D), silu(h @ w["v"].T).view(T, H, E)
    o = torch.stack([lightning_steps(q[:, a], k[:, a], v[:, a], m["decay"][a]) for a in range(H)], 1).reshape(T, H * E)
    return (rms_norm(o, w["norm"], eps) * torch.sigmoid(h @ w["g"].T)) @ w["o"].T


def side_by_side(h, w, m, eps):
    return m["left_scale"] * head_normed_attention(h, sub(w, "left."), m["left"], eps) + \
        m["right_scale"] * lightning_attention(h, sub(w, "right."), m["right"], eps)


def gated_ff(h, w):
    return (silu(h @ w["gate"].T) * (h @ w["up"].T)) @ w["down"].T


def relu_squared_ff(h, up, down):
    return torch.clamp(h @ up.T, min=0) ** 2 @ down.T


def choose_experts(s, router):
    """(ids [T, top], margin [T]): the `top` largest scores among the experts of the best groups; a group's score is the sum
    of its two largest. The margin is the smallest distance at which either choice would turn."""
    T, X = s.shape
    groups = router.get("groups") or {"count": 1, "keep": 1}
    n, keep, top = groups["count"], groups["keep"], router["top"]
    size = X // n
    group_score = torch.topk(s.view(T, n, size), min(2, size), dim=-1).values.sum(-1)
    kept = torch.topk(group_score, keep, dim=-1).indices
    allowed = torch.zeros(T, n, dtype=torch.bool).scatter(-1, kept, True).repeat_interleave(size, -1)
    masked = s.masked_fill(~allowed, -math.inf)
    best = torch.topk(masked, min(top + 1, X), dim=-1)
    margin = torch.full((T,), math.inf, dtype=s.dtype)
    if top < keep * size:
        margin = best.values[:, top - 1] - best.values[:, top]
    if keep < n:
        edge = torch.topk(group_score, keep + 1, dim=-1).values
        margin = torch.minimum(margin, edge[:, keep - 1] - edge[:, keep])
    return best.indices[:, :top], margin


def routed_ff(h, w, mlp, margins=None):
    router = mlp["router"]
    s = torch.sigmoid(h @ w["router"].T)
    ids, margin = choose_experts(s, router)
    if margins is not None:
        margins.append(margin)
    out = torch.zeros_like(h)
    for e in range(router["experts"]):
        rows = torch.nonzero((ids == e).any(-1)).flatten()
        if len(rows):
            y = relu_squared_ff(h[rows], w[f"e{e}.up"], w[f"e{e}.down"])
            out[rows] = out[rows] + router["scale"] * s[rows, e, None] * y
    if mlp.get("shared"):
        out = out + relu_squared_ff(h, w["shared.up"], w["shared.down"])
    return out


def sub(weights, prefix):
    """The tensors whose names start with `prefix`, by the rest of their names."""
    return {k[len(prefix):]: v for k, v in weights.items() if k.startswith(prefix)}


def forward(config, weights, tokens, dtype=torch.float64, layers_out=None, margins=None):
    """Logits [T, V] of a whole sequence. weights: name -> tensor (any float type). layers_out: a list that gets the
    stream after every layer; margins: a list that gets every routed layer's choice margin per token."""
    w = {k: (v.to(dtype) if v.is_floating_point() else v) for k, v in weights.items()}
    eps = config["norm"]["eps"]

    def norm(x, name):
        return layer_norm(x, w[name], w[name + ".b"], eps)
    x = w["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    held = {}
    for i, layer in enumerate(config["layers"]):
        p, m, mix = f"l{i}.", layer["mixer"], sub(w, f"l{i}.mix.")
        h = norm(x, p + "norm1")
        if layer["type"] == "parallel":
            y = side_by_side(h, mix, m, eps)
        elif layer["type"] == "attention":
            y = whole_normed_attention(h, mix, m, eps)
        else:
            if m.get("kv_from") is None:
                held[i] = chunked_keys_values(h, mix, m)
            y = differential_attention(h, mix, m, eps, held[m["kv_from"] if m.get("kv_from") is not None else i])
        x = x + norm(y, p + "norm1b")
        if layer.get("mlp") is not None:
            h, ff = norm(x, p + "norm2"), sub(w, p + "mlp.")
            y = gated_ff(h, ff) if layer["mlp"]["kind"] == "dense" else routed_ff(h, ff, layer["mlp"], margins)
            x = x + norm(y, p + "norm2b")
        if layers_out is not None:
            layers_out.append(x.clone())
    return norm(x, "final.norm") @ w["head"].T
