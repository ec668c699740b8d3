"""The kernels of polarquant_amd.latent_ops, each against the plain float64 implementation."""
import math

import pytest
import torch

from oracle import dekipel_oracle as do
from polarquant_amd import _ffi
from polarquant_amd import latent_ops as ops

pytestmark = pytest.mark.gpu
DT = {"f32": torch.float32, "bf16": torch.bfloat16, "f16": torch.float16}
TOL = {"f32": 3e-6, "bf16": 6e-3, "f16": 8e-4}         # error over the largest magnitude of the result


def err(got, want):
    return float((got.double().cpu() - want).abs().max() / want.abs().max())


def rand(g, *shape, dt="f32", s=1.0):
    return (torch.randn(shape, generator=g) * s).to(DT[dt])


# ---------------------------------------------------------------- norms and convolution
@pytest.mark.parametrize("width,groups,taps", [(w, n, t) for w, n in ((96, 3), (70, 14), (250, 2), (512, 1), (1024, 4), (2560, 5)) for t in (1, 2, 4, 5, 9)]
                         + [(w, n, t) for w, n in ((4096, 4), (5120, 1), (4096, 128), (8192, 2)) for t in (4, 5)])
def test_norm_conv(gpu, width, groups, taps):
    g = torch.Generator().manual_seed(width + taps)
    for dt in ("f32", "bf16", "f16"):
        for L in (1, 3, 32, 33, 75):
            B = 2
            x, y = rand(g, B, L, width), rand(g, B, L, width, dt=dt, s=3.0)
            wpost, wpre = 1 + rand(g, width, s=0.3).to(DT[dt]), 1 + rand(g, width, s=0.3).to(DT[dt])
            cw = rand(g, width, taps, dt=dt, s=0.5)
            hist = rand(g, B, max(taps - 1, 0), width)
            st = ops.ConvState(B, taps, width, gpu)
            st.rows.copy_(hist)
            xs, h = ops.norm_conv(x.to(gpu), wpre.to(gpu), groups, 1e-4, y.to(gpu), wpost.to(gpu), cw.to(gpu), st)
            for b in range(B):
                xw = x[b].double() + do.grouped_rms_norm(y[b].double(), wpost.double(), 1e-4, groups)
                n = torch.cat([hist[b].double(), do.grouped_rms_norm(xw, wpre.double(), 1e-4, groups)])
                hw = do.input_conv(n, cw.double())[-L:]
                assert err(xs[b], xw) < 3e-6 and err(h[b], hw) < TOL[dt], (dt, L, b)
                if taps > 1:
                    assert err(st.rows[b], n[-(taps - 1):]) < 3e-6, (dt, L, b)
            _, plain = ops.norm_conv(x.to(gpu), wpre.to(gpu), groups, 1e-4)
            assert err(plain[0], do.grouped_rms_norm(x[0].double(), wpre.double(), 1e-4, groups)) < TOL[dt]


def test_norm_conv_portions_give_the_same_bits(gpu):
    """Strips recompute what lies before them, portions read it from the state: neither may show."""
    g = torch.Generator().manual_seed(7)
    W, taps, L = 640, 4, 200
    x, y, cw = rand(g, 1, L, W).to(gpu), rand(g, 1, L, W, dt="bf16").to(gpu), rand(g, W, taps, dt="bf16").to(gpu)
    w = (1 + rand(g, W, s=0.2)).bfloat16().to(gpu)

    def run(cuts):
        st, outs, at = ops.ConvState(1, taps, W, gpu), [], 0
        for n in cuts:
            xo, h = ops.norm_conv(x[:, at:at + n].clone(), w, 2, 1e-5, y[:, at:at + n].contiguous(), w, cw, st)
            outs.append((xo, h))
            at += n
        assert at == L
        return torch.cat([o[0] for o in outs], 1), torch.cat([o[1] for o in outs], 1), st.rows.clone()
    whole = run([L])
    for cuts in ([1] * 5 + [2] + [L - 7], [33, 64, 100, 3], [32] * 6 + [8], [2] * 100, [199, 1]):
        for a, b in zip(whole, run(cuts)):
            assert torch.equal(a, b), cuts


def test_norm_conv_left_padding(gpu):
    """Tokens before a sequence's start leave no trace in the convolution."""
    g = torch.Generator().manual_seed(8)
    W, taps = 96, 4
    start = torch.tensor([0, 3, 39, 40], dtype=torch.int32)
    x, cw, w = rand(g, 4, 60, W), rand(g, W, taps), 1 + rand(g, W, s=0.2)
    st = ops.ConvState(4, taps, W, gpu)
    h = []
    for a, b in ((0, 2), (2, 41), (41, 42), (42, 60)):       # starts before, inside and at the edges of portions
        h.append(ops.norm_conv(x[:, a:b].contiguous().to(gpu), w.to(gpu), 3, 1e-5, conv_w=cw.to(gpu), state=st, start=start.to(gpu), pos=a)[1])
    h = torch.cat(h, 1)
    for b, s in enumerate(start.tolist()):
        want = do.input_conv(do.grouped_rms_norm(x[b, s:].double(), w.double(), 1e-5, 3), cw.double())
        assert err(h[b, s:], want) < 3e-6 and not h[b, :s].any(), b


# ---------------------------------------------------------------- latents' norms, elementwise, products
@pytest.mark.parametrize("q_rank,kv_rank,extra", [(64, 96, 128), (18, 36, 5), (11, 13, 0), (1536, 512, 64), (7, 1, 3)])
def test_latent_norm(gpu, q_rank, kv_rank, extra):
    g = torch.Generator().manual_seed(q_rank)
    for dt, L in [(dt, L) for dt in DT for L in (5, 401)]:        # few tokens: a workgroup each, many: a wavefront each
        B, pos = 3, 9
        p = rand(g, B, L, q_rank + kv_rank + extra, dt=dt, s=2.0)
        wq, wc = (1 + rand(g, q_rank, s=0.3)).to(DT[dt]), (1 + rand(g, kv_rank, s=0.3)).to(DT[dt])
        cache = torch.full((B, L + 15, kv_rank), 7.0, dtype=DT[dt], device=gpu)
        cq = ops.latent_norm(p.to(gpu), wq.to(gpu), wc.to(gpu), cache, 1e-3, pos)
        assert err(cq, do.rms_norm(p[..., :q_rank].double(), wq.double(), 1e-3)) < TOL[dt]
        assert err(cache[:, pos:pos + L], do.rms_norm(p[..., q_rank:q_rank + kv_rank].double(), wc.double(), 1e-3)) < TOL[dt]
        assert bool((cache[:, :pos] == 7).all()) and bool((cache[:, pos + L:] == 7).all())
        assert torch.equal(ops.latent_norm(p.to(gpu), wq.to(gpu), None, None, 1e-3, pos), cq)
        again = torch.zeros_like(cache)
        ops.latent_norm(p.to(gpu), wq.to(gpu), wc.to(gpu), again, 1e-3, 0, torch.tensor([pos], dtype=torch.int32, device=gpu))
        assert torch.equal(again[:, pos:pos + L], cache[:, pos:pos + L])


@pytest.mark.parametrize("n", [1, 8, 13, 4096, 100003])
def test_relu_sq(gpu, n):
    g = torch.Generator().manual_seed(n)
    for dt in DT:
        x = rand(g, n, dt=dt)
        x[0] = 1.5
        assert err(ops.relu_sq(x.to(gpu)), x.double().clamp(min=0) ** 2) < TOL[dt]


@pytest.mark.parametrize("heads,N,K", [(1, 256, 512), (7, 96, 64), (3, 48, 32), (5, 64, 96), (2, 512, 128), (3, 20, 12), (1, 7, 13), (2, 16, 8192)])
def test_head_linear(gpu, heads, N, K):
    g = torch.Generator().manual_seed(N + K)
    for dt in DT:
        for M in (1, 3, 8, 9, 16, 37):
            x, w = rand(g, M, heads, K, dt=dt), rand(g, heads, N, K, dt=dt, s=K ** -0.5)
            wide = rand(g, M, heads * N + 24, dt=dt)
            gate = wide[:, 8:8 + heads * N]
            want = torch.einsum("mhk,hnk->mhn", x.double(), w.double())
            xg, wg = x.to(gpu), w.to(gpu)
            assert err(ops.head_linear(xg, wg), want) < TOL[dt], (dt, M)
            assert err(ops.head_linear(xg, wg, epilogue=_ffi.PQ_EPI_RELU_SQ), want.clamp(min=0) ** 2) < TOL[dt]
            f32 = ops.head_linear(xg, wg, epilogue=_ffi.PQ_EPI_F32)
            assert f32.dtype == torch.float32 and err(f32, want) < 5e-6
            gated = ops.head_linear(xg, wg, gate=wide.to(gpu)[:, 8:8 + heads * N])
            assert err(gated, want * torch.sigmoid(gate.double()).view(M, heads, N)) < TOL[dt]


# ---------------------------------------------------------------- attention over the latents
def decode_want(q, c, sink, scale, pos, start):
    B, L, H, R = q.shape
    out = torch.zeros(B, L, H, R, dtype=torch.float64)
    for b in range(B):
        k = c[b, :pos + L].double()[:, None].expand(-1, H, -1)
        out[b] = do.attend(q[b].double(), k, k, sink.double(), scale, int(start[b]) if start is not None else 0).view(L, H, R)
    return out


@pytest.mark.parametrize("R", [64, 96, 128, 200, 256, 320, 512, 8, 520, 37])
@pytest.mark.parametrize("L,H", [(1, 1), (1, 16), (1, 17), (3, 20), (1, 40), (2, 64), (16, 7)])
def test_latent_decode(gpu, R, L, H):
    g = torch.Generator().manual_seed(R * 131 + L * 7 + H)
    lengths = {1: (0, 31, 32, 127), 2: (100,), 3: (61, 300), 16: (15,)}[L]
    for dt in ("bf16", "f16", "f32"):
        for pos in lengths:
            B, cap = 2, pos + L + 40
            q, c = rand(g, B, L, H, R, dt=dt, s=2.0), rand(g, B, cap, R, dt=dt)
            # one key far back stands out for the last query of head 0: a lost key shows
            c[0, (pos + L) // 3] = q[0, -1, 0] * 0.7
            sink = rand(g, H, s=2.0)
            start = None if pos < 40 else torch.tensor([0, 37], dtype=torch.int32)
            want = decode_want(q, c, sink, R ** -0.5, pos, start)
            for S in (1, 2, 5):
                got = ops.latent_decode_attention(q.to(gpu), c.to(gpu), sink.to(gpu), R ** -0.5, pos, start=None if start is None else start.to(gpu), n_splits=S)
                assert err(got, want) < {"f32": 5e-6, "bf16": 1.2e-2, "f16": 2e-3}[dt], (dt, pos, S)


def test_latent_decode_positions_in_device_memory_and_stale_rows(gpu):
    """Rows past the sequence hold large finite values from an earlier use; the position comes from the device."""
    g = torch.Generator().manual_seed(3)
    for dt in ("bf16", "f32"):
        for pos in (0, 63, 64, 500):
            q, c, sink = rand(g, 2, 1, 24, 128, dt=dt), rand(g, 2, 640, 128, dt=dt), rand(g, 24)
            c[:, pos + 1:] = 3e4
            dev = torch.tensor([pos], dtype=torch.int32, device=gpu)
            got = ops.latent_decode_attention(q.to(gpu), c.to(gpu), sink.to(gpu), 0.1, 0, dev, n_splits=9)
            assert err(got, decode_want(q, c, sink, 0.1, pos, None)) < (1.2e-2 if dt == "bf16" else 5e-6), (dt, pos)


def test_latent_decode_sink_and_first_tokens(gpu):
    """A sink far above every score leaves almost nothing of the values, one far below leaves the plain softmax; the first
    token of a sequence is a key like any other."""
    g = torch.Generator().manual_seed(4)
    q, c = rand(g, 1, 1, 16, 64, dt="bf16"), rand(g, 1, 256, 64, dt="bf16")
    c[0, 0] = q[0, 0, 3] * 1.5
    for level in (-60.0, 0.0, 8.0, 60.0):
        sink = torch.full((16,), level)
        want = decode_want(q, c, sink, 0.3, 200, None)
        got = ops.latent_decode_attention(q.to(gpu), c.to(gpu), sink.to(gpu), 0.3, 200, n_splits=3).cpu().double()
        assert float((got - want).abs().max()) <= 1.2e-2 * float(want.abs().max()) + 1e-12, level
        assert bool(torch.isfinite(got).all())
    assert float(want.abs().max()) < 1e-10


@pytest.mark.parametrize("D,Dv", [(64, 64), (64, 40), (40, 24), (128, 128), (96, 112), (192, 128), (136, 7), (256, 256), (8, 200)])
def test_latent_prefill(gpu, D, Dv):
    g = torch.Generator().manual_seed(D + Dv)
    H = 3
    for dt in ("bf16", "f16"):
        for L, past in ((17, 0), (64, 0), (130, 0), (65, 63), (33, 200), (20, 1)):
            B, Lk = 2, past + L
            ld = -(-Lk // 64) * 64
            q, k, v = rand(g, B, L, H, D, dt=dt), rand(g, B, Lk, H, D, dt=dt), rand(g, B, Lk, H, Dv, dt=dt)
            far = max(0, Lk // 2 - 1)
            k[0, far, 1] = q[0, -1, 1] * 1.2
            k[1, 0, 2] = q[1, -1, 2] * 1.2                      # the first token
            sink, scale = rand(g, H, s=2.0), 1.5 * D ** -0.5
            start = torch.tensor([0, min(70, Lk - 1) if past == 0 and L > 100 else 0], dtype=torch.int32)
            vt = torch.full((B, H, Dv, ld), 1e4, dtype=DT[dt])
            vt[..., :Lk] = v.permute(0, 2, 3, 1)
            wide = rand(g, B * L, H * Dv + 16, dt=dt)
            gate = wide[:, 8:8 + H * Dv]
            got = ops.latent_prefill_attention(q.to(gpu), k.to(gpu), vt.to(gpu), sink.to(gpu), scale, wide.to(gpu)[:, 8:8 + H * Dv], start.to(gpu))
            bare = ops.latent_prefill_attention(q.to(gpu), k.to(gpu), vt.to(gpu), sink.to(gpu), scale)
            for b in range(B):
                s = int(start[b])
                full = do.attend_fast(q[b].double(), k[b].double(), v[b].double(), sink.double(), scale)
                assert err(bare[b], full) < {"bf16": 1.2e-2, "f16": 2e-3}[dt], (dt, L, past, b)
                if s:
                    full = do.attend(q[b].double(), k[b].double(), v[b].double(), sink.double(), scale, s)
                want = full * torch.sigmoid(gate[b * L:(b + 1) * L].double())
                assert err(got[b], want) < {"bf16": 1.2e-2, "f16": 2e-3}[dt], (dt, L, past, b)
