"""Small Darolix configurations and weights made for testing.

The configurations differ from each other in every size, in the order of their layers, in what the loop runs and in what
the design allows to be absent, equal or one (a layer without a feed-forward, no identity experts, all experts chosen, one
expert, one head, one key head for all heads and one for each, one group or one a head, a norm in one part or in parts that
straddle heads, a convolution of one tap, no soft cap, no temperature or one that steps at every token, values larger and
smaller than keys, a loop over one layer, over all and none, sizes that are no multiples of 16, 8 or 4). Weights are drawn
so that every path matters: norm weights away from one, slow and fast decays (a lost state shows hundreds of tokens later),
router rows that spread the tokens over the experts, corrections that change the choice, skips away from zero.
"""
from __future__ import annotations

import math

import torch

from kanavik_util import Driver, row_error, write_folder  # noqa: F401  (the same driver of the package's step function)


def mamba2(heads, vdim, state, groups, conv, norm_groups, mlp=None):
    m = {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "conv": conv, "norm_groups": norm_groups}
    return {"type": "mamba2", "mixer": m, "mlp": mlp}


def parallel(left, right, mlp=None):
    return {"type": "parallel", "mixer": {"left": left, "right": right}, "mlp": mlp}


def left(heads, kv_heads, dim, vdim, scale, softcap=None, coef=None, every=None):
    d = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if softcap:
        d["softcap"] = softcap
    if coef is not None:
        d["q_temp"] = {"coef": coef, "every": every}
    return d


def right(heads, dim, vdim, tau):
    return {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau}


def moe(experts, identity, top, ff):
    return {"kind": "moe", "router": {"experts": experts, "identity": identity, "top": top}, "expert": {"ff": ff}}


def config(layers, width, vocab, scale=4.0, loop=None, eps=1e-5):
    c = {"architecture": "Darolix", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": scale},
         "layers": layers}
    if loop:
        c["loop"] = dict(zip(("start", "stop", "times"), loop))
    return c


# sizes that are no multiples of 16; a parallel layer first, values smaller than keys, a temperature that steps at every
# token; one group a head and norm parts that straddle heads; layers 1 .. 2 run three times
CONFIG_ODD = config([parallel(left(6, 3, 24, 20, 0.2, 8.0, 0.5, 1), right(3, 20, 24, 8.0), mlp=moe(5, 2, 3, 40)),
                     mamba2(6, 10, 21, 6, 3, 4, mlp=moe(3, 1, 1, 24)),
                     parallel(left(4, 1, 18, 34, 0.3, None, 0.2, 50), right(1, 13, 10, 1.0)),
                     mamba2(4, 20, 12, 2, 4, 1)],
                    width=88, vocab=211, scale=9.4, loop=(1, 3, 3))
# a state-space layer first and last; many experts; keys and values of 64, one key head per head; a key size of 128 and
# states of 100; all experts chosen, no identities; a convolution of one tap; the whole model runs twice
CONFIG_WIDE = config([mamba2(8, 32, 100, 1, 4, 8, mlp=moe(16, 8, 4, 64)),
                      parallel(left(8, 8, 32, 64, 0.15, 20.0, 0.4, 7), right(2, 128, 64, 16.0), mlp=moe(4, 0, 4, 32)),
                      mamba2(2, 96, 16, 2, 1, 3, mlp=moe(1, 3, 2, 48))],
                     width=128, vocab=300, scale=11.0, loop=(0, 3, 2), eps=1e-6)
# one layer, run as it stands; sizes that are no multiples of 4
CONFIG_ONE = config([parallel(left(2, 2, 14, 6, 0.4), right(2, 9, 7, 4.0))], width=50, vocab=97, scale=1.0)

CONFIGS = {"odd": CONFIG_ODD, "wide": CONFIG_WIDE, "one": CONFIG_ONE}
RANKS = {"odd": 5, "wide": 70, "one": 1}                # of the decays: no key of config.json, a tensor's shape


def tensor_shapes(c, rank=16):
    """Names and shapes of a checkpoint, written from the design's naming and not from the package's parts."""
    C = c["width"]
    shapes = {"embed": (c["vocab"], C), "head": (c["vocab"], C), "final.norm": (C,)}
    for i, lay in enumerate(c["layers"]):
        p, m = f"l{i}.", lay["mixer"]
        shapes[p + "norm1"] = (C,)
        q = p + "mix."
        if lay["type"] == "mamba2":
            H, inner = m["heads"], m["heads"] * m["vdim"]
            ch = inner + 2 * m["groups"] * m["state"]
            shapes.update({q + "in": (inner + ch + H, C), q + "conv": (ch, m["conv"]), q + "conv.b": (ch,), q + "dt_bias": (H,),
                           q + "A_log": (H,), q + "D": (H,), q + "norm": (inner,), q + "o": (C, inner)})
        else:
            a, b = m["left"], m["right"]
            H, G, D, E = a["heads"], a["kv_heads"], a["dim"], a["vdim"]
            shapes.update({q + "left.q": (H * D, C), q + "left.k": (G * D, C), q + "left.v": (G * E, C), q + "left.o": (C, H * E),
                           q + "left.out": (C,), q + "right.out": (C,)})
            H, D, E = b["heads"], b["dim"], b["vdim"]
            shapes.update({q + "right.q": (H * D, C), q + "right.k": (H * D, C), q + "right.v": (H * E, C), q + "right.g": (H * E, C),
                           q + "right.o": (C, H * E), q + "right.norm": (E,), q + "right.a1": (rank, C),
                           q + "right.a2": (H * D, rank), q + "right.a2.b": (H * D,)})
        if lay["mlp"]:
            q, F = p + "mlp.", lay["mlp"]["expert"]["ff"]
            router = lay["mlp"]["router"]
            n = router["experts"] + router.get("identity", 0)
            shapes[q + "router"], shapes[q + "correction"] = (n, C), (n,)
            for e in range(router["experts"]):
                shapes.update({q + f"e{e}.gate": (F, C), q + f"e{e}.up": (F, C), q + f"e{e}.down": (C, F)})
    return shapes


def make_weights(c, seed, rank=16, sharp=1.0):
    """{name: bfloat16 tensor}: what a checkpoint of configuration C holds. SHARP > 1 makes a key match its own query far
    better than others do: the rows of each query head become those of its key head where their sizes agree."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(c, rank).items():
        leaf = name.split(".")[-1]
        normal = torch.randn(shape, generator=g)
        if name == "embed":
            t = normal
        elif leaf in ("norm1", "norm", "out"):
            t = 1.0 + 0.3 * normal
        elif leaf == "conv":
            t = 0.6 * normal
        elif leaf == "b" and ".a2." in name:
            t = 3.0 + 2.0 * normal                                 # decays of 0.5 to 0.999
        elif leaf == "b":
            t = 0.3 * normal
        elif leaf == "dt_bias":
            t = -2.0 + normal                                      # step sizes of 0.05 to 0.3
        elif leaf == "A_log":
            t = normal - 0.5
        elif leaf == "D":
            t = 0.7 * normal
        elif leaf == "router":
            t = 2.5 * normal / math.sqrt(shape[-1])
        elif leaf == "correction":
            t = 0.2 * normal
        else:                                                      # linear maps [out, in]
            t = normal / math.sqrt(shape[-1])
        out[name] = t.to(torch.bfloat16)
    if sharp > 1.0:
        for i, lay in enumerate(c["layers"]):
            if lay["type"] == "parallel":
                a, p = lay["mixer"]["left"], f"l{i}.mix.left."
                per = a["heads"] // a["kv_heads"]
                k = out[p + "k"].view(a["kv_heads"], a["dim"], -1)
                q = out[p + "q"].view(a["heads"], a["dim"], -1)
                for h in range(a["heads"]):
                    q[h] = k[h // per]
    return out
