"""The latent-attention decoder beside the closest existing model of this package (the Llama shell with the polar-key
cache) at equal width, heads, feed-forward work and layers; random weights, bf16.

    python -m polarquant_amd.benchmarks.latent_bench [--kernels] [--models] [--sizes large medium] [--context 16384] [--batch 8]

--kernels: each kernel of the latent path against its bound, beside the like kernel of the other model, timed as captured
graphs of back-to-back calls over rotated buffers (more than the 256 MB last-level cache where it streams).
--models: prompt and decode throughput of both models, the decode step replayed from its HIP graph.
"""
from __future__ import annotations

import argparse
import json
import math
import time

import torch
import torch.nn.functional as F

from .. import _ffi
from .. import latent_ops as ops
from ..modeling_dekipel import DekipelConfig, DekipelForCausalLM, DekipelLayerConfig, LatentMixerConfig
from .linear_bench import _graph_time_us

HBM, MFMA = 8e12, 2.5e15            # bytes/s, dense bf16 flop/s

# width, heads (query), KV heads of the Llama shell, ff of its gated feed-forward, ranks; head dimension 128 throughout.
# The squared-relu feed-forward has two matrices of 1.5 times that ff: the same weights and work.
SIZES = {"large": dict(width=4096, heads=32, kv_heads=8, ff=14336, q_rank=1536, kv_rank=512),
         "medium": dict(width=2048, heads=16, kv_heads=8, ff=8192, q_rank=768, kv_rank=256)}
VOCAB = 32768


def dekipel_config(s, layers, capacity=0, share=2):
    """Every `share`-th layer owns its latent, the others read the one before."""
    out = []
    for i in range(layers):
        m = LatentMixerConfig(s["heads"], 128, 128, s["q_rank"], s["kv_rank"], 128 ** -0.5, None if i % share == 0 else i - i % share)
        out.append(DekipelLayerConfig(m, s["ff"] * 3 // 2))
    return DekipelConfig(VOCAB, s["width"], out, 1e-5, 4, 4, cache_capacity=capacity)


def build_dekipel(s, layers, dev, dtype=torch.bfloat16, share=2):
    torch.manual_seed(0)
    prev = torch.get_default_dtype()
    torch.set_default_dtype(dtype)
    try:
        with torch.device(dev):
            m = DekipelForCausalLM(dekipel_config(s, layers, share=share))
    finally:
        torch.set_default_dtype(prev)
    g = torch.Generator(device=dev).manual_seed(1)
    with torch.no_grad():
        for p in m.parameters():
            if p.dim() == 2:
                p.normal_(0.0, 1.0 / math.sqrt(p.shape[1]) if p.shape[1] > 16 else 0.3, generator=g)
    return m.eval()


def _line(kernel, us, nbytes, flops, like=None):
    bound = max(nbytes / HBM, flops / MFMA) * 1e6
    out = {"kernel": kernel, "us": round(us, 2), "bytes": int(nbytes), "flops": int(flops), "bound": "hbm" if nbytes / HBM >= flops / MFMA else "mfma",
           "frac_of_bound": round(bound / us, 4)}
    if like:
        out["like"] = like
        out["times_as_far"] = round(like["frac_of_bound"] / out["frac_of_bound"], 3)
    return out


def kernels(s, B, ctx, emit):
    dev, dt = torch.device("cuda:0"), torch.bfloat16
    H, R, W, Q = s["heads"], s["kv_rank"], s["width"], s["q_rank"]
    D = Dv = 128
    r = lambda *shape: torch.randn(*shape, device=dev, dtype=torch.float32).to(dt)

    # ---- decode
    for b, n in ((B, ctx), (1, ctx * 8)):
        nbuf = max(2, int(600e6 // (b * n * R * 2)) + 1)
        cs = [r(b, n, R) for _ in range(nbuf)]
        q, sink = r(b, 1, H, R), torch.zeros(H, device=dev)
        us = _graph_time_us(lambda i: ops.latent_decode_attention(q, cs[i], sink, 0.05, n - 1), nbuf)
        nb = b * n * R * 2 + 2 * q.numel() * 2
        fl = 4 * b * n * H * R
        del cs
        like = polar_attention_like(s, b, n)
        emit(_line("latent_decode_kernel + merge, batch %d x %d keys" % (b, n), us, nb, fl, like))
    M = B
    for name, heads, N, K, gated in (("queries to the latent space", H, R, D, False), ("latent output to the heads, gated", H, Dv, R, True)):
        nbuf = int(600e6 // (heads * N * K * 2)) + 1
        ws, x, gate = [r(heads, N, K) for _ in range(nbuf)], r(M, heads, K), r(M, heads * N)
        us = _graph_time_us(lambda i: ops.head_linear(x, ws[i], gate if gated else None), nbuf)
        emit(_line("head_linear (%s), %d rows" % (name, M), us, heads * N * K * 2, 2 * M * heads * N * K, small_linear_like(heads * N // 4, K * 4, M)))      # the like kernel with as many weight bytes
    for name, N, K, act in (("input projections", Q + R + H * Dv, W, 0), ("query up", H * D, Q, 0), ("output", W, H * Dv, 0), ("feed-forward up", s["ff"] * 3 // 2, W, 1),
                            ("feed-forward down", W, s["ff"] * 3 // 2, 0)):
        nbuf = int(600e6 // (N * K * 2)) + 1
        ws, x = [r(N, K) for _ in range(nbuf)], r(M, K)
        us = _graph_time_us(lambda i: ops.linear(x, ws[i], relu_squared=bool(act)), nbuf)
        emit(_line("linear (%s), %d rows" % (name, M), us, N * K * 2, 2 * M * N * K))
    state = ops.ConvState(M, 4, W, dev)
    x, y, w, cw = torch.randn(M, 1, W, device=dev), r(M, 1, W), r(W), r(W, 4)
    us = _graph_time_us(lambda i: ops.norm_conv(x, w, 4, 1e-5, y, w, cw, state), 50)
    from ..decode_ops import rmsnorm
    xh = r(M, 1, W)
    us2 = _graph_time_us(lambda i: rmsnorm(xh, w, 1e-5, residual=y, sum_out=xh), 50)
    emit(_line("norm_conv, %d rows (latency)" % M, us, M * W * 36, 0, dict(_line("rmsnorm, %d rows (latency)" % M, us2, M * W * 8, 0))))
    p, cache = r(M, 1, Q + R + H * Dv), r(M, 64, R)
    r_q, r_c = r(Q), r(R)
    us = _graph_time_us(lambda i: ops.latent_norm(p, r_q, r_c, cache, 1e-5, 3), 50)
    emit(_line("latent_norm, %d rows (latency)" % M, us, M * (Q + R) * 4, 0))

    # ---- prompt
    L = ctx
    q, k, gate = r(1, L, H, D), r(1, L, H, D), r(L, H * Dv)
    vt, sink = r(1, H, Dv, L), torch.zeros(H, device=dev)
    us = _graph_time_us(lambda i: ops.latent_prefill_attention(q, k, vt, sink, 0.08, gate), 4)
    fl = L * L * H * (D + Dv)
    q4, k4, v4 = r(1, H, L, D), r(1, s["kv_heads"], L, D), r(1, s["kv_heads"], L, D)
    us2 = _graph_time_us(lambda i: F.scaled_dot_product_attention(q4, k4, v4, is_causal=True, enable_gqa=True), 4)
    emit(_line("latent_prefill_kernel, %d tokens" % L, us, 4 * L * H * D * 2, fl, _line("scaled_dot_product_attention, causal", us2, 0, fl)))
    del q, k, gate, vt, q4, k4, v4
    x, y = torch.randn(1, L, W, device=dev), r(1, L, W)
    state = ops.ConvState(1, 4, W, dev)
    us = _graph_time_us(lambda i: ops.norm_conv(x, w, 4, 1e-5, y, w, cw, state), 8)
    xh = r(1, L, W)
    us2 = _graph_time_us(lambda i: rmsnorm(xh, w, 1e-5, residual=y, sum_out=xh), 8)
    emit(_line("norm_conv, %d tokens" % L, us, L * W * 12, 0, _line("rmsnorm + residual", us2, L * W * 8, 0)))
    p, cache = r(1, L, Q + R + H * Dv), r(1, L, R)
    us = _graph_time_us(lambda i: ops.latent_norm(p, r_q, r_c, cache, 1e-5, 0), 8)
    emit(_line("latent_norm, %d tokens" % L, us, L * (Q + R) * 4, 0, _line("rmsnorm + residual", us2, L * W * 8, 0)))
    from ..decode_ops import silu_mul
    a, b2 = r(L, s["ff"] * 3 // 2), r(L, s["ff"] * 3 // 2)
    us = _graph_time_us(lambda i: ops.relu_sq(a), 4)
    us2 = _graph_time_us(lambda i: silu_mul(a, b2), 4)
    emit(_line("relu_sq, %d tokens" % L, us, a.numel() * 4, 0, _line("silu_mul", us2, a.numel() * 6, 0)))


def small_linear_like(N, K, M):
    from ..decode_ops import linear_small_m
    nbuf = int(600e6 // (N * K * 2)) + 1
    ws = [torch.randn(N, K, device="cuda:0", dtype=torch.bfloat16) for _ in range(nbuf)]
    x = torch.randn(M, K, device="cuda:0", dtype=torch.bfloat16)
    us = _graph_time_us(lambda i: linear_small_m(x, ws[i]), nbuf)
    return _line("linear_small_m [%d, %d]" % (N, K), us, N * K * 2, 2 * M * N * K)


def polar_attention_like(s, B, n):
    """The polar-key decode attention at the same heads, batch and context (4/4-bit codes, bf16 values)."""
    from ..attention import polar_decode_attention
    dev, dt, Nk, N = torch.device("cuda:0"), torch.bfloat16, s["kv_heads"], s["heads"]
    g = n // 128
    nbuf = max(2, int(600e6 // (B * n * Nk * 324)) + 1)
    r = lambda *shape: torch.randn(*shape, device=dev, dtype=torch.float32).to(dt)
    sets = [(torch.randint(0, 256, (B, Nk, g, 128, 64), dtype=torch.uint8, device=dev), [r(B, Nk, g, 1, 64).abs() * 0.1 for _ in range(4)],
             r(B, Nk, 128, 128), r(B, Nk, g * 128 + 1, 128)) for _ in range(nbuf)]
    q = r(B, N, 1, 128)
    us = _graph_time_us(lambda i: polar_decode_attention(q, sets[i][0], *sets[i][1], sets[i][2], sets[i][3], g, 1), nbuf)
    return _line("polar_decode_attention (pair kernel + merge), %d KV heads" % Nk, us, B * Nk * n * 324, 4 * B * n * N * 128)


def _throughput(name, model, decoder, B, L, new, layers):
    dev = torch.device("cuda:0")
    ids = torch.randint(0, VOCAB, (B, L), generator=torch.Generator(device=dev).manual_seed(3), device=dev)
    decoder.prefill(ids)                                      # (library initialisation, allocator)
    torch.cuda.synchronize()
    t0 = time.perf_counter()
    tok = decoder.prefill(ids).argmax(-1)
    torch.cuda.synchronize()
    t_p = time.perf_counter() - t0
    tok = decoder.step(tok).argmax(-1)                        # captures
    torch.cuda.synchronize()
    t0 = time.perf_counter()
    for _ in range(new):
        tok = decoder.step(tok).argmax(-1)
    torch.cuda.synchronize()
    t_d = (time.perf_counter() - t0) / new
    return {"model": name, "layers": layers, "batch": B, "prompt": L, "prefill_tokens_per_s": round(B * L / t_p, 1), "prefill_ms": round(t_p * 1e3, 2),
            "decode_ms_per_step": round(t_d * 1e3, 4), "decode_tokens_per_s": round(B / t_d, 1), "cache_bytes_per_token": model.kv_cache_bytes_per_token(),
            "parameters": sum(p.numel() for p in model.parameters()), "peak_memory_GiB": round(torch.cuda.max_memory_allocated() / 2 ** 30, 2)}


def models(s, B, L, emit, layers=4, new=64, which=("dekipel", "llama_polar")):
    from ..graph_decode import LayeredGraphDecoder, PolarGraphDecoder
    from ..modeling_common import PolarConfig
    from .e2e_bench import build_model
    dev = torch.device("cuda:0")
    out = {}
    with torch.no_grad():
        if "dekipel" in which:
            torch.cuda.reset_peak_memory_stats()
            m = build_dekipel(s, layers, dev)
            out["dekipel"] = _throughput("dekipel", m, LayeredGraphDecoder(m, L + new + 128), B, L, new, layers)
            emit(out["dekipel"])
            del m
            torch.cuda.empty_cache()
        if "llama_polar" in which:
            torch.cuda.reset_peak_memory_stats()
            m = build_model(PolarConfig(hidden_size=s["width"], num_attention_heads=s["heads"], num_key_value_heads=s["kv_heads"], num_hidden_layers=layers,
                                        intermediate_size=s["ff"], vocab_size=VOCAB, eos_token_id=[VOCAB + 1]), dev)
            out["llama_polar"] = _throughput("llama_polar", m, PolarGraphDecoder(m, L + new + 128, fused_prefill=True), B, L, new, layers)
            emit(out["llama_polar"])
            del m
            torch.cuda.empty_cache()
    return out


def run(sizes, B, ctx, want_kernels, want_models, emit):
    for name in sizes:
        tag = lambda d: emit(dict({"size": name}, **d))
        if want_kernels:
            kernels(SIZES[name], B, ctx, tag)
            torch.cuda.empty_cache()
        if want_models:
            models(SIZES[name], B, ctx, tag)
            models(SIZES[name], 1, ctx, tag)


def main(argv=None):
    ap = argparse.ArgumentParser(description=__doc__.split("\n\n")[0])
    ap.add_argument("--kernels", action="store_true")
    ap.add_argument("--models", action="store_true")
    ap.add_argument("--sizes", nargs="+", choices=sorted(SIZES), default=["large", "medium"])
    ap.add_argument("--context", type=int, default=16384)
    ap.add_argument("--batch", type=int, default=8)
    a = ap.parse_args(argv)
    both = not (a.kernels or a.models)
    run(a.sizes, a.batch, a.context, a.kernels or both, a.models or both, lambda d: print(json.dumps(d), flush=True))


if __name__ == "__main__":
    main()
