"""Small Dekipel configurations with random weights, written as checkpoint directories, for the tests."""
import json
import os

import torch
from safetensors.torch import save_file

from oracle import dekipel_oracle as do


def layer(heads, dim, vdim, q_rank, kv_rank, scale, ff, kv_from=None):
    m = {"heads": heads, "dim": dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank, "scale": scale}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": m, "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def config(width, vocab, layers, groups=1, taps=3, eps=1e-6):
    return {"architecture": "Dekipel", "width": width, "vocab": vocab, "canon": {"taps": taps}, "norm": {"eps": eps, "groups": groups},
            "layers": layers}


# sizes the matrix-core kernels take throughout; a shared latent, a layer without feed-forward, layers of different shapes
EVEN = config(192, 256, [layer(4, 32, 64, 64, 96, 0.2, 256), layer(9, 64, 32, 96, 128, 0.11, None), layer(5, 32, 32, 64, 96, 0.3, 128, kv_from=0),
                         layer(4, 64, 32, 64, 128, 0.125, 320, kv_from=1)], groups=3, taps=3)
# awkward sizes: nothing is a multiple of anything useful, one head, norm groups of 14 channels, seven taps
ODD = config(70, 101, [layer(3, 20, 12, 18, 36, 0.25, 90), layer(1, 7, 10, 11, 13, 0.4, 33), layer(2, 24, 5, 40, 36, 0.2, None, kv_from=0)],
             groups=5, taps=7, eps=1e-2)
# one tap: no state at all; ranks a multiple of 8 but not of 32, head sizes that need a padded tile
PADDED = config(160, 144, [layer(6, 40, 24, 48, 40, 0.16, 200), layer(6, 72, 56, 56, 72, 0.12, 64)], groups=2, taps=1)
ALL = {"even": EVEN, "odd": ODD, "padded": PADDED}


def write(path, cfg, seed, dtype=torch.bfloat16, weights=None):
    """-> the weights of the checkpoint directory it writes."""
    w = weights if weights is not None else do.random_weights(cfg, seed, dtype)
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file(w, os.path.join(path, "model.safetensors"))
    return w


def tokens(n, vocab, seed):
    return torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def rel_rms(got, want):
    """Root mean square of the difference over that of `want`, the worst row."""
    got, want = got.double().cpu(), want.double()
    return float(((got - want).pow(2).mean(-1).sqrt() / want.pow(2).mean(-1).sqrt()).max())
