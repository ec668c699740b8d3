"""Dekipel models of random shapes, prompts cut at random, against the plain implementation."""
import random

import pytest
import torch

from oracle import dekipel_oracle as do
from polarquant_amd.checkpoint import load_pretrained

import dekipel_cases as dc

pytestmark = pytest.mark.gpu


def random_config(r: random.Random):
    step = r.choice([1, 4, 8, 16, 32])                     # what the sizes are multiples of
    size = lambda lo, hi: max(1, -(-r.randint(lo, hi) // step)) * step
    groups = r.choice([1, 2, 3, 4, 6])
    width = groups * size(24, 300 // groups + 24)
    layers, owners = [], []
    for i in range(r.randint(1, 5)):
        rank = size(5, 200)
        src = r.choice(owners) if owners and r.random() < 0.4 else None
        if src is not None:
            rank = layers[src]["mixer"]["kv_rank"]
        else:
            owners.append(i)
        dim = size(4, 140)
        layers.append(dc.layer(r.randint(1, 18), dim, size(3, 140), size(5, 120), rank, r.uniform(0.5, 2.0) * dim ** -0.5,
                               None if r.random() < 0.15 else size(20, 300), src))
    return dc.config(width, size(20, 300), layers, groups, r.randint(1, 6), r.choice([1e-6, 1e-5, 1e-2]))


@pytest.mark.parametrize("seed", range(12))
def test_random_model(gpu, tmp_path, seed):
    r = random.Random(seed)
    cfg = random_config(r)
    w = dc.write(str(tmp_path), cfg, seed)
    n = r.randint(40, 260)
    t = dc.tokens(n, cfg["vocab"], seed)
    cuts, left = [], n
    while left:
        cuts.append(min(left, r.choice([1, 1, 2, 3, 16, 17, 31, 32, 33, 64, 65, r.randint(1, n)])))
        left -= cuts[-1]
    want = do.forward(t, cfg, w)
    for dtype in (torch.float32, torch.bfloat16):
        model = load_pretrained(str(tmp_path), dtype, gpu)
        whole = model(input_ids=torch.tensor([t], device=gpu)).logits[0]
        past, got, at = None, [], 0
        for c in cuts:
            out = model(input_ids=torch.tensor([t[at:at + c]], device=gpu), past_key_values=past)
            past, at = out.past_key_values, at + c
            got.append(out.logits[0])
        for name, lg in (("whole", whole), ("portions", torch.cat(got))):
            d = lg.double().cpu() - want
            err = d.pow(2).mean(-1).sqrt() / want.pow(2).mean(-1).sqrt()
            # 16-bit: a row now and then is badly conditioned (a small norm group that nearly vanishes), so the mean is what binds
            if dtype == torch.float32:
                assert float(err.max()) < 2e-4 and float(err.mean()) < 1e-5, (name, cfg, cuts)
            else:
                assert float(err.mean()) < 4e-2 and float(err.median()) < 4e-2, (name, cfg, cuts)
