"""The Kapudra decoder (windowed attention beside a gated delta rule, matrix memories) beside the closest existing models of this
package at equal width, heads, feed-forward work and layers: the Dekipel decoder (kernels) and the Llama shell with the
polar-key cache (whole models); random weights, bf16.

    python -m polarquant_amd.benchmarks.recurrent_bench [--kernels] [--models] [--sizes large medium] [--context 16384] [--batch 8]

--kernels: each kernel against its bound, beside the like kernel of the other model, timed as captured graphs of back-to-back
calls over rotated buffers (more than the 256 MB last-level cache where it streams).
--models: prompt and decode throughput of both models, the decode step replayed from its HIP graph.
"""
from __future__ import annotations

import argparse
import json
import math

import torch
import torch.nn.functional as F

from .. import layer_ops
from .. import latent_ops
from .. import recurrent_ops as ops
from ..modeling_kapudra import (DeltaMixerConfig, KapudraConfig, KapudraForCausalLM, KapudraLayerConfig, MemoryMixerConfig, ParallelMixerConfig,
                                WindowMixerConfig)
from ..modeling_recurrent import MemoryState
from ..recurrent_ops import Step
from .latent_bench import HBM, MFMA, VOCAB, _line, _throughput, small_linear_like
from .linear_bench import _graph_time_us

# width, query heads (delta-rule heads alike), KV heads, ff; head dimension 128 throughout; heads of the matrix memories (128 x 256)
SIZES = {"large": dict(width=4096, heads=32, kv_heads=8, ff=14336, window=2048, memory_heads=16, rank=128),
         "medium": dict(width=2048, heads=16, kv_heads=8, ff=8192, window=1024, memory_heads=8, rank=64)}


def kapudra_config(s, layers):
    """Parallel and matrix-memory layers in turn."""
    par = ParallelMixerConfig(WindowMixerConfig(s["heads"], s["kv_heads"], 128, 128, s["window"], 128 ** -0.5),
                              DeltaMixerConfig(s["heads"], s["heads"], 128, 128, 4, s["rank"], s["rank"]), 0.7, 0.7)
    mem = MemoryMixerConfig(s["memory_heads"], 128, 256, 15.0)
    return KapudraConfig(VOCAB, s["width"], [KapudraLayerConfig(mem if i % 2 else par, s["ff"]) for i in range(layers)], 1e-5, math.sqrt(s["width"]), 1.0, 30.0)


def build_kapudra(s, layers, dev, dtype=torch.bfloat16):
    torch.manual_seed(0)
    prev = torch.get_default_dtype()
    torch.set_default_dtype(dtype)
    try:
        with torch.device(dev):
            m = KapudraForCausalLM(kapudra_config(s, layers))
    finally:
        torch.set_default_dtype(prev)
    g = torch.Generator(device=dev).manual_seed(1)
    with torch.no_grad():
        for p in m.parameters():
            if p.dim() == 2:
                p.normal_(0.0, 1.0 / math.sqrt(p.shape[1]) if p.shape[1] > 16 else 0.5, generator=g)
    return m.eval()


def kernels(s, B, ctx, emit):
    dev, dt = torch.device("cuda:0"), torch.bfloat16
    H, G, W, D, window, MH, MV = s["heads"], s["kv_heads"], s["width"], 128, s["window"], s["memory_heads"], 256
    r = lambda *shape: torch.randn(*shape, device=dev, dtype=torch.float32).to(dt)
    f = lambda *shape: torch.randn(*shape, device=dev, dtype=torch.float32)
    slopes = torch.tensor([2.0 ** (-8.0 * (h + 1) / H) for h in range(H)], device=dev)

    def delta_inputs(M):
        return ops.DeltaInputs(r(M, H * D), r(M, H * D), r(M, H * D), f(M, H).abs() * 0.01, f(M, H).abs() * 0.1, -f(M, H * D).abs() * 0.1, torch.rand(M, H, device=dev))

    # ---- decode
    pos = 4 * window + 5
    for b in (B, 1):
        step = Step(b, 1, pos)
        nbuf = max(2, int(600e6 // (b * G * window * D * 4)) + 1)
        rings = [ops.WindowRing(b, G, D, D, window, dt, dev) for _ in range(nbuf)]
        for x in rings:
            x.k.normal_(), x.v.normal_()
        q, out = r(b, H * D), torch.empty(b, H * D, dtype=dt, device=dev)
        us = _graph_time_us(lambda i: ops.window_attention(q, rings[i], slopes, D ** -0.5, step, out), nbuf)
        like = latent_decode_like(s, b, 2 * window * G * D // 512)
        emit(_line("window_attention, batch %d x %d keys" % (b, window), us, b * G * window * D * 4 + 4 * q.numel(), 4 * b * window * H * D, like))
        del rings
        nbuf = max(2, int(600e6 // (b * H * D * D * 8)) + 1)
        states, x = [torch.zeros(b, H, D, D, device=dev) for _ in range(nbuf)], delta_inputs(b)
        us = _graph_time_us(lambda i: ops.delta_scan(x, states[i], step), nbuf)
        emit(_line("delta_scan, batch %d" % b, us, b * H * D * D * 8, 8 * b * H * D * D, latent_decode_like(s, b, H * D * D * 8 // 1024)))
        nbuf = max(2, int(600e6 // (b * MH * D * MV * 8)) + 1)
        states = [MemoryState(b, MH, D, MV, dev) for _ in range(nbuf)]
        p, li, lf = r(b, 2 * MH * D + MH * MV), f(b, MH), -f(b, MH).abs()
        us = _graph_time_us(lambda i: ops.memory_scan(p[:, :MH * D], p[:, MH * D:2 * MH * D], p[:, 2 * MH * D:], li, lf, states[i].S, states[i].m, 0.1, step), nbuf)
        emit(_line("memory_scan, batch %d" % b, us, b * MH * D * (MV + 1) * 8, 5 * b * MH * D * MV, latent_decode_like(s, b, MH * D * MV * 8 // 1024)))
        del states
    M, step = B, Step(B, 1, pos)
    from ..decode_ops import rmsnorm, silu_mul
    w, xh, y = r(W), r(M, 1, W), r(M, 1, W)
    norm_like = lambda m, xx, yy, n: _line("rmsnorm + residual, %d rows" % m, _graph_time_us(lambda i: rmsnorm(xx, w, 1e-5, residual=yy, sum_out=xx), n), m * W * 8, 0)
    few = norm_like(M, xh, y, 50)
    xs = f(M, 1, W)
    us = _graph_time_us(lambda i: layer_ops.norm_conv(xs, w, 1, 1e-5, y), 50)
    emit(_line("norm_conv (plain residual), %d rows (latency)" % M, us, M * W * 12, 0, few))
    proj, ring = r(M, (H + 2 * G) * D), ops.WindowRing(M, G, D, D, window, dt, dev)
    wq, wk = r(H * D), r(G * D)
    us = _graph_time_us(lambda i: ops.qk_norm(proj[:, :H * D], proj[:, H * D:(H + G) * D], proj[:, (H + G) * D:], wq, wk, H, 1e-5, ring, step), 50)
    emit(_line("qk_norm + append, %d rows (latency)" % M, us, proj.numel() * 4, 0, few))
    dp = delta_prep_args(s, M, r, dev)
    us = _graph_time_us(lambda i: ops.delta_prep(*dp, step), 50)
    emit(_line("delta_prep, %d rows (latency)" % M, us, M * H * D * 20, 0, few))
    o, gate, nw, out = f(M, H * D), r(M, H * D), r(D), torch.empty(M, H * D, dtype=dt, device=dev)
    us = _graph_time_us(lambda i: ops.head_norm_gate(o, nw, gate, H, 1e-5, out), 50)
    emit(_line("head_norm_gate, %d rows (latency)" % M, us, M * H * D * 8, 0, few))
    a, b2 = r(M, s["ff"]), r(M, s["ff"])
    act = _line("silu_mul, %d rows" % M, _graph_time_us(lambda i: silu_mul(a, b2), 50), a.numel() * 6, 0)
    us = _graph_time_us(lambda i: layer_ops.gelu_mul(a, b2), 50)
    emit(_line("gelu_mul, %d rows (latency)" % M, us, a.numel() * 6, 0, act))
    n_par = (H + 2 * G) * D + 3 * H * D + 2 * s["rank"] + H + 2 * s["ff"]
    n_mem = 2 * MH * D + 2 * MH * MV + 16 + 2 * s["ff"]
    for name, N, K in (("input projections, parallel layer", n_par // 16 * 16, W), ("output projections, parallel layer", W, 2 * H * D + s["ff"]),
                       ("input projections, matrix memory", n_mem // 16 * 16, W), ("output projections, matrix memory", W, MH * MV + s["ff"])):
        nbuf = int(600e6 // (N * K * 2)) + 1
        ws, x = [r(N, K) for _ in range(nbuf)], r(M, K)
        us = _graph_time_us(lambda i: layer_ops.linear(x, ws[i]), nbuf)
        emit(_line("linear (%s), %d rows" % (name, M), us, N * K * 2, 2 * M * N * K, small_linear_like(N, K, M)))
        del ws
    for name, N, K in (("decay or gate up", H * D, s["rank"]),):
        nbuf = int(600e6 // (N * K * 2)) + 1
        ws, x = [r(N, K) for _ in range(nbuf)], r(M, K)
        us = _graph_time_us(lambda i: layer_ops.linear(x, ws[i]), nbuf)
        emit(_line("linear (%s), %d rows" % (name, M), us, N * K * 2, 2 * M * N * K, small_linear_like(N // 4, K * 4, M)))
        del ws

    # ---- prompt
    L, step = ctx, Step(1, ctx, 0)
    q4, k4, v4 = r(1, H, L, D), r(1, G, L, D), r(1, G, L, D)
    sdpa = _line("scaled_dot_product_attention, causal", _graph_time_us(lambda i: F.scaled_dot_product_attention(q4, k4, v4, is_causal=True, enable_gqa=True), 4), 0,
                 2 * L * L * H * D)
    ql, vt, sink = r(1, L, H, D), r(1, H, D, L), torch.zeros(H, device=dev)
    like = _line("latent_prefill_kernel, causal", _graph_time_us(lambda i: latent_ops.latent_prefill_attention(ql, ql, vt, sink, 0.08), 4), 4 * L * H * D * 2, 2 * L * L * H * D)
    emit(dict(sdpa))
    del q4, k4, v4, vt
    q, kn, vn, out = ql.view(L, H * D), r(L, G * D), r(L, G * D), torch.empty(L, H * D, dtype=dt, device=dev)
    ring = ops.WindowRing(1, G, D, D, window, dt, dev)
    us = _graph_time_us(lambda i: ops.window_attention(q, ring, slopes, D ** -0.5, step, out, 1.0, kn, vn), 4)
    keys = window * (L - window) + window * (window + 1) // 2
    emit(_line("window_attention, %d tokens, window %d" % (L, window), us, L * (2 * H + 2 * G) * D * 2, 4 * keys * H * D, like))
    del ql, q, kn, vn, out
    x = delta_inputs(L)
    S = torch.zeros(1, H, D, D, device=dev)
    us = _graph_time_us(lambda i: ops.delta_scan(x, S, step), 2)
    emit(_line("delta_scan, %d tokens" % L, us, L * H * D * (6 + 4 + 4), 8 * L * H * D * D, like))
    del x
    p, li, lf, st = r(L, 2 * MH * D + MH * MV), f(L, MH), -f(L, MH).abs(), MemoryState(1, MH, D, MV, dev)
    us = _graph_time_us(lambda i: ops.memory_scan(p[:, :MH * D], p[:, MH * D:2 * MH * D], p[:, 2 * MH * D:], li, lf, st.S, st.m, 0.1, step), 2)
    emit(_line("memory_scan, %d tokens" % L, us, p.numel() * 2 + L * MH * MV * 4, 4 * L * MH * D * MV, like))
    del p
    xh, y, xs = r(1, L, W), r(1, L, W), f(1, L, W)
    many = norm_like(L, xh, y, 8)
    us = _graph_time_us(lambda i: layer_ops.norm_conv(xs, w, 1, 1e-5, y), 8)
    emit(_line("norm_conv (plain residual), %d tokens" % L, us, L * W * 12, 0, many))
    proj = r(L, (H + 2 * G) * D)
    us = _graph_time_us(lambda i: ops.qk_norm(proj[:, :H * D], proj[:, H * D:(H + G) * D], proj[:, (H + G) * D:], wq, wk, H, 1e-5, ring, step), 8)
    emit(_line("qk_norm, %d tokens" % L, us, L * (H + G) * D * 4, 0, many))
    dp = delta_prep_args(s, L, r, dev)
    us = _graph_time_us(lambda i: ops.delta_prep(*dp, step), 4)
    emit(_line("delta_prep, %d tokens" % L, us, L * H * D * (3 * 4 + 2 + 4), 0, many))
    del dp
    o, gate, out = f(L, H * D), r(L, H * D), torch.empty(L, H * D, dtype=dt, device=dev)
    us = _graph_time_us(lambda i: ops.head_norm_gate(o, nw, gate, H, 1e-5, out), 8)
    emit(_line("head_norm_gate, %d tokens" % L, us, L * H * D * 8, 0, many))
    a, b2, out = r(L, s["ff"]), r(L, s["ff"]), torch.empty(L, s["ff"], dtype=dt, device=dev)
    act = _line("silu_mul", _graph_time_us(lambda i: silu_mul(a, b2), 4), a.numel() * 6, 0)
    us = _graph_time_us(lambda i: layer_ops.gelu_mul(a, b2, out), 4)
    emit(_line("gelu_mul, %d tokens" % L, us, a.numel() * 6, 0, act))


def delta_prep_args(s, M, r, dev):
    H, D = s["heads"], 128
    p = r(M, 3 * H * D + H)
    B = M if M < 64 else 1
    return (p[:, :H * D], p[:, H * D:2 * H * D], p[:, 2 * H * D:3 * H * D], p[:, 3 * H * D:], r(M, H * D), r(H * D, 4), r(H * D, 4), r(H * D, 4), r(H), r(H * D),
            layer_ops.ConvState(B, 4, 3 * H * D, dev), D, D)


def latent_decode_like(s, B, n):
    """The latent decode attention over a cache of as many bytes: n keys of rank 512 per sequence."""
    dev, dt = torch.device("cuda:0"), torch.bfloat16
    n = max(64, n // 64 * 64)
    nbuf = max(2, int(600e6 // (B * n * 1024)) + 1)
    r = lambda *shape: torch.randn(*shape, device=dev, dtype=torch.float32).to(dt)
    cs, q, sink = [r(B, n, 512) for _ in range(nbuf)], r(B, 1, s["heads"], 512), torch.zeros(s["heads"], device=dev)
    us = _graph_time_us(lambda i: latent_ops.latent_decode_attention(q, cs[i], sink, 0.05, n - 1), nbuf)
    return _line("latent_decode_kernel + merge, batch %d x %d keys" % (B, n), us, B * n * 1024 + 4 * q.numel(), 4 * B * n * s["heads"] * 512)


def models(s, B, L, emit, layers=4, new=64, which=("kapudra", "llama_polar")):
    from .latent_bench import models as other_models
    dev = torch.device("cuda:0")
    if "kapudra" in which:
        with torch.no_grad():
            torch.cuda.reset_peak_memory_stats()
            m = build_kapudra(s, layers, dev)
            line = _throughput("kapudra", m, m.graph_decoder(L + new + 128), B, L, new, layers)
            emit(dict(line, state_bytes_per_sequence=m.state_bytes()))
            del m
            torch.cuda.empty_cache()
    rest = [x for x in which if x != "kapudra"]
    if rest:
        other_models(s, B, L, emit, layers, new, rest)


def run(sizes, B, ctx, want_kernels, want_models, emit, which=("kapudra", "llama_polar")):
    for name in sizes:
        tag = lambda d: emit(dict({"size": name}, **d))
        if want_kernels:
            kernels(SIZES[name], B, ctx, tag)
            torch.cuda.empty_cache()
        if want_models:
            models(SIZES[name], B, ctx, tag, which=which)
            models(SIZES[name], 1, ctx, tag, which=which)


def main(argv=None):
    ap = argparse.ArgumentParser(description=__doc__.split("\n\n")[0])
    ap.add_argument("--kernels", action="store_true")
    ap.add_argument("--models", action="store_true")
    ap.add_argument("--sizes", nargs="+", choices=sorted(SIZES), default=["large", "medium"])
    ap.add_argument("--which", nargs="+", choices=("kapudra", "llama_polar"), default=["kapudra", "llama_polar"])
    ap.add_argument("--context", type=int, default=16384)
    ap.add_argument("--batch", type=int, default=8)
    a = ap.parse_args(argv)
    both = not (a.kernels or a.models)
    run(a.sizes, a.batch, a.context, a.kernels or both, a.models or both, lambda d: print(json.dumps(d), flush=True), a.which)


if __name__ == "__main__":
    main()
