"""Small Kapudra configurations with random weights for the tests."""
import json

import torch

import dekipel_cases as dc
from oracle import kapudra_oracle as ko

tokens, rel_rms = dc.tokens, dc.rel_rms


def close(got, want, limit):
    """Every row within the limit in float32; in 16 bits all but the few in which a matrix memory's normalizer, near zero, takes
    the other sign with the rounding (always possible at a sequence's first token, when it is one product), and the typical
    row well within it."""
    got, want = got.double().cpu(), want.double()
    off = ((got - want).pow(2).mean(-1).sqrt() / want.pow(2).mean(-1).sqrt()).flatten()
    if limit < 1e-3:
        return float(off.max()) < limit
    return int((off > limit).sum()) <= 3 + off.numel() // 25 and float(off.median()) < limit / 3


def parallel(left, right, left_scale, right_scale, ff):
    """left: heads, kv_heads, dim, vdim, window, scale; right: heads, kv_heads, dim, vdim, conv."""
    a, r = dict(zip(("heads", "kv_heads", "dim", "vdim"), left)), dict(zip(("heads", "kv_heads", "dim", "vdim", "conv"), right))
    a.update(mask={"size": left[4]}, scale=left[5])
    return {"type": "parallel", "mixer": {"left": a, "right": r, "left_scale": left_scale, "right_scale": right_scale},
            "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def memory(heads, dim, vdim, cap, ff):
    return {"type": "mlstm", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": cap}, "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def config(width, vocab, layers, loop=None, eps=1e-6, embedding=3.0, logit_scale=0.7, softcap=3.0):
    return {"architecture": "Kapudra", "width": width, "vocab": vocab, "layers": layers, "norm": {"eps": eps}, "embedding": {"scale": embedding},
            "logit_scale": logit_scale, "logit_softcap": softcap, "loop": None if loop is None else dict(zip(("start", "stop", "times"), loop))}


# sizes the matrix-core kernels take; grouped heads on both sides, a layer without feed-forward, three passes over the middle
EVEN = config(160, 208, [parallel((4, 2, 32, 64, 40, 0.3), (4, 2, 32, 48, 3), 0.5, 1.2, 224), memory(3, 16, 40, 7.0, 96),
                         parallel((6, 1, 64, 32, 75, 0.2), (2, 2, 64, 32, 4), 1.1, 0.4, None), memory(2, 64, 24, 15.0, None)], (1, 3, 3))
# nothing is a multiple of anything useful, a long filter, a loop that begins the model
ODD = config(70, 101, [parallel((3, 1, 20, 12, 7, 0.4), (3, 1, 7, 10, 7), 0.8, 0.9, 33), memory(5, 9, 6, 4.0, 21), memory(1, 13, 20, 9.0, None),
                       parallel((2, 2, 5, 18, 33, 0.5), (1, 1, 18, 5, 2), 1.3, 0.7, 50)], (0, 2, 2), eps=1e-2, embedding=1.0, softcap=6.0)
# ones: a window of the token itself, a filter of one tap, single heads, one pass over all layers
ONES = config(96, 144, [memory(1, 32, 32, 10.0, 64), parallel((1, 1, 16, 16, 1, 1.0), (1, 1, 16, 16, 1), 1.0, 1.0, 32)], (0, 2, 1), logit_scale=1.0)
# wide heads, no loop
WIDE = config(256, 160, [parallel((2, 1, 136, 128, 130, 0.1), (2, 1, 128, 128, 4), 0.65, 0.85, 288), memory(1, 200, 136, 11.0, 128)])
ALL = {"even": EVEN, "odd": ODD, "ones": ONES, "wide": WIDE}
RANKS = {"even": (40, 16), "odd": (5, 11), "ones": (1, 3), "wide": (64, 32)}


def weights(cfg, seed, ranks=(12, 20), dtype=torch.bfloat16):
    return ko.random_weights(cfg, seed, dtype, decay_rank=ranks[0], gate_rank=ranks[1])


def write(path, cfg, seed, ranks=(12, 20), w=None):
    """-> the weights of the checkpoint directory it writes."""
    return dc.write(path, cfg, 0, weights=w if w is not None else weights(cfg, seed, ranks))


def changed(cfg, f):
    c = json.loads(json.dumps(cfg))
    f(c)
    return c
