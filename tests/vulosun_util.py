"""Small Vulosun configurations and weights made for testing.

The configurations differ from each other in every size, in the order of their layers, in who reads whose keys and values and
in what the design allows to be absent, equal or one (a layer without a feed-forward, no shared expert, one group, groups of one
expert, all groups kept, all experts chosen, one expert, one head, one key head for all heads and one for each, a chunk of one
position, of less than a page and of more than any sequence, two readers of one layer's pages with chunks of their own, a
rotation of two elements and of the whole head, a scaling or none, decays of one and of almost nothing, values larger and smaller
than keys, sizes that are no multiples of 16, 8 or 4). Weights are drawn so that every path matters: norm weights away from
one and biases away from zero, sinks of any sign, lambdas that subtract much, slow and fast decays (a lost state shows hundreds
of tokens later), router rows that spread the tokens over the experts.
"""
from __future__ import annotations

import math

import torch

from kanavik_util import Driver, row_error, write_folder  # noqa: F401  (the same driver of the package's step function)


def rot(base, dims, factor=None):
    return {"base": base, "dims": dims, **({"scaling": {"factor": factor}} if factor is not None else {})}


def attention(heads, kv_heads, dim, vdim, scale, rot, mlp=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "rot": rot}
    return {"type": "attention", "mixer": m, "mlp": mlp}


def differential(heads, kv_heads, dim, vdim, scale, rot, chunk, diff, mlp=None, kv_from=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "rot": rot, "mask": {"size": chunk}, "diff": diff}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "attention_2", "mixer": m, "mlp": mlp}


def left(heads, kv_heads, dim, vdim, scale, rot):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "rot": rot}


def right(heads, dim, vdim, decay):
    return {"heads": heads, "dim": dim, "vdim": vdim, "decay": decay}


def parallel(left, right, left_scale=0.8, right_scale=0.5, mlp=None):
    return {"type": "parallel", "mixer": {"left": left, "right": right, "left_scale": left_scale, "right_scale": right_scale}, "mlp": mlp}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff, scale=1.0, groups=None, shared=None):
    router = {"experts": experts, "top": top, "scale": scale}
    if groups:
        router["groups"] = dict(zip(("count", "keep"), groups))
    return {"kind": "moe", "router": router, "expert": {"ff": ff}, **({"shared": {"ff": shared}} if shared else {})}


def config(layers, width, vocab, eps=1e-5):
    return {"architecture": "Vulosun", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}


# sizes that are no multiples of 16; a chunk of 10 positions whose pages two later layers read, one with chunks of 17, one with
# 6; values smaller than two maps; groups of one expert; a parallel layer last, without a feed-forward
R_ODD = rot(700.0, 6, 2.5)
CONFIG_ODD = config([differential(6, 3, 11, 20, 0.3, R_ODD, 10, 0.25, mlp=moe(6, 2, 40, 1.7, (6, 4), 24)),
                     attention(6, 2, 24, 34, 0.2, rot(1e4, 10), mlp=dense(72)),
                     differential(6, 3, 11, 20, 0.25, R_ODD, 17, 0.6, mlp=moe(8, 3, 20, 0.5, (2, 1)), kv_from=0),
                     differential(6, 3, 11, 20, 0.4, R_ODD, 6, 0.1, mlp=moe(5, 5, 24, 2.0, None, 40), kv_from=0),
                     parallel(left(6, 3, 22, 14, 0.35, rot(500.0, 22)), right(3, 20, 24, [0.3, 1.0, 0.97]), 1.3, 0.7)],
                    width=88, vocab=211)
# a parallel layer first, attention last; keys and values of 64 and 128 with one key head per head and one for all; a chunk longer
# than any sequence, no scaling; 64 experts in 8 groups; two differential layers with pages of their own
CONFIG_WIDE = config([parallel(left(4, 4, 64, 64, 0.15, rot(1e5, 32)), right(2, 128, 64, [0.9, 0.999]), -0.6, 1.1, mlp=moe(64, 4, 64, 2.5, (8, 3), 96)),
                      differential(8, 1, 32, 64, 0.2, rot(1e4, 32), 1000, 0.4, mlp=moe(12, 2, 32, 1.0, (3, 3), 64)),
                      differential(2, 2, 64, 128, 0.12, rot(5e4, 2), 32, 0.3, mlp=dense(200)),
                      attention(8, 2, 32, 16, 0.3, rot(1e6, 32), mlp=moe(1, 1, 48, 0.3, None, 16))],
                     width=128, vocab=300, eps=1e-6)
# one layer without a feed-forward; sizes that are no multiples of 4
CONFIG_ONE = config([parallel(left(2, 1, 14, 6, 0.4, rot(100.0, 4)), right(1, 9, 7, [0.8]))], width=50, vocab=97)

CONFIGS = {"odd": CONFIG_ODD, "wide": CONFIG_WIDE, "one": CONFIG_ONE}


def attention_shapes(q, m, C, maps=1):
    H, G, D, E = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    return {q + "q": (H * maps * D, C), q + "k": (G * maps * D, C), q + "v": (G * E, C), q + "o": (C, H * E)}


def tensor_shapes(c):
    """Names and shapes of a checkpoint, written from the design's naming and not from the package's parts."""
    C = c["width"]
    shapes = {"embed": (c["vocab"], C), "head": (c["vocab"], C), "final.norm": (C,), "final.norm.b": (C,)}
    for i, lay in enumerate(c["layers"]):
        p, m = f"l{i}.", lay["mixer"]
        for name in ("norm1", "norm1b") + (("norm2", "norm2b") if lay["mlp"] else ()):
            shapes[p + name] = shapes[p + name + ".b"] = (C,)
        q = p + "mix."
        if lay["type"] == "parallel":
            a, b = m["left"], m["right"]
            shapes.update(attention_shapes(q + "left.", a, C))
            shapes.update({q + "left.q.norm": (a["dim"],), q + "left.k.norm": (a["dim"],), q + "left.sink": (a["heads"],)})
            H, D, E = b["heads"], b["dim"], b["vdim"]
            shapes.update({q + "right.q": (H * D, C), q + "right.k": (H * D, C), q + "right.v": (H * E, C), q + "right.g": (H * E, C),
                           q + "right.o": (C, H * E), q + "right.norm": (H * E,)})
        elif lay["type"] == "attention":
            shapes.update(attention_shapes(q, m, C))
            shapes.update({q + "q.norm": (m["heads"] * m["dim"],), q + "k.norm": (m["kv_heads"] * m["dim"],), q + "g": (m["heads"], C)})
        else:
            own = attention_shapes(q, m, C, maps=2)
            own.update({name + ".b": shape[:1] for name, shape in own.items() if name != q + "o"})
            if m.get("kv_from") is not None:
                own = {name: shape for name, shape in own.items() if name[len(q)] not in "kv"}
            shapes.update(own)
            shapes.update({q + "g": (m["heads"], C), **{q + n: (m["dim"],) for n in ("lq1", "lk1", "lq2", "lk2")}})
        if lay["mlp"]:
            q, mlp = p + "mlp.", lay["mlp"]
            if mlp["kind"] == "dense":
                shapes.update({q + "gate": (mlp["ff"], C), q + "up": (mlp["ff"], C), q + "down": (C, mlp["ff"])})
                continue
            n, F = mlp["router"]["experts"], mlp["expert"]["ff"]
            shapes[q + "router"] = (n, C)
            for e in range(n):
                shapes.update({q + f"e{e}.up": (F, C), q + f"e{e}.down": (C, F)})
            if mlp.get("shared"):
                shapes.update({q + "shared.up": (mlp["shared"]["ff"], C), q + "shared.down": (C, mlp["shared"]["ff"])})
    return shapes


def make_weights(c, seed, sharp=1.0):
    """{name: bfloat16 tensor}: what a checkpoint of configuration C holds. SHARP > 1 makes a key match its own query far
    better than others do: the rows of each query head (and map) become those of its key head, SHARP times as large."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(c).items():
        leaf = name.split(".")[-1]
        normal = torch.randn(shape, generator=g)
        if name == "embed":
            t = 2.0 * normal
        elif leaf in ("norm1", "norm1b", "norm2", "norm2b", "norm"):
            t = 1.0 + 0.3 * normal
        elif leaf == "b" and ".mix." in name:
            t = 0.4 * normal
        elif leaf == "b":
            t = 0.3 * normal
        elif leaf == "sink":
            t = 1.5 * normal
        elif leaf in ("lq1", "lk1", "lq2", "lk2"):
            t = 0.8 * normal / math.sqrt(math.sqrt(shape[0]))
        elif leaf == "router":
            t = 2.5 * normal / math.sqrt(shape[-1])
        else:                                                      # linear maps [out, in]
            t = normal / math.sqrt(shape[-1])
        out[name] = t.to(torch.bfloat16)
    if sharp > 1.0:
        for i, lay in enumerate(c["layers"]):
            m, maps = lay["mixer"], 2 if lay["type"] == "attention_2" else 1
            a, p = (m["left"], f"l{i}.mix.left.") if lay["type"] == "parallel" else (m, f"l{i}.mix.")
            if p + "k" not in out:
                continue
            per = a["heads"] // a["kv_heads"]
            k = out[p + "k"].view(a["kv_heads"], maps * a["dim"], -1)
            out[p + "q"] = (sharp * k.repeat_interleave(per, 0).reshape(a["heads"] * maps * a["dim"], -1).float()).to(torch.bfloat16)
    return out
