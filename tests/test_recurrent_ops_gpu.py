"""The kernels of polarquant_amd.recurrent_ops and the layer steps of the Kapudra decoder, each against the plain float64
implementation."""
import math

import pytest
import torch

from oracle import kapudra_oracle as ko
from polarquant_amd import layer_ops
from polarquant_amd import recurrent_ops as ops
from polarquant_amd.recurrent_ops import Step

pytestmark = pytest.mark.gpu
DT = {"f32": torch.float32, "bf16": torch.bfloat16, "f16": torch.float16}
TOL = {"f32": 1e-5, "bf16": 1e-2, "f16": 2e-3}         # error over the largest magnitude of the result


def err(got, want):
    return float((got.double().cpu() - want).abs().max() / want.abs().max())


def rand(g, *shape, dt="f32", s=1.0):
    return (torch.randn(shape, generator=g) * s).to(DT[dt])


def cut(n, sizes):
    out, at, i = [], 0, 0
    while at < n:
        out.append(min(sizes[i % len(sizes)], n - at))
        at += out[-1]
        i += 1
    return out


# ---------------------------------------------------------------- elementwise
def test_elementwise_steps(gpu):
    g = torch.Generator().manual_seed(0)
    for dt in DT:
        for M, n, pad in ((1, 5, 3), (7, 64, 0), (130, 1032, 8), (3, 257, 1)):
            wide = rand(g, M, 2 * n + pad, dt=dt, s=2.0)
            out = torch.zeros(M, n + 2 * pad, dtype=DT[dt], device=gpu)
            w = wide.to(gpu)
            layer_ops.gelu_mul(w[:, :n], w[:, n + pad:], out[:, pad:pad + n])
            assert err(out[:, pad:pad + n], ko.gelu_tanh(wide[:, :n].double()) * wide[:, n + pad:].double()) < TOL[dt]
            assert float(out[:, :pad].abs().sum() + out[:, pad + n:].abs().sum()) == 0
            x, e, y, v = rand(g, M, n), rand(g, M, n), rand(g, M, n, dt=dt), rand(g, n, dt=dt)
            for yy, ee, vv in ((y, e, v), (None, e, v), (y, None, None), (None, None, v)):
                dev = lambda t: None if t is None else t.to(gpu)
                got = layer_ops.stream_add(dev(x), dev(yy), dev(ee), dev(vv))
                want = x.double() + sum(t.double() for t in (yy, ee, vv) if t is not None)
                assert err(got, want) < 1e-6
            _, h = layer_ops.norm_conv(x.to(gpu).view(1, M, n), v.to(gpu), 1, 1e-3, y.to(gpu).view(1, M, n))     # plain residual add
            assert err(h[0], ko.rms_norm(x.double() + y.double(), v.double(), 1e-3)) < TOL[dt]
            table = rand(g, 19, n, dt=dt)
            ids = torch.randint(0, 19, (2, M), generator=g)
            assert err(layer_ops.embed_rows(table.to(gpu), ids.to(gpu), 3.25), table[ids].double() * 3.25) < 1e-6
    z = rand(g, 3, 500, s=20.0)
    assert err(layer_ops.softcap(z.clone().to(gpu), 0.5, 8.0), ko.cap(z.double() * 0.5, 8.0)) < 1e-6
    assert err(layer_ops.softcap(z.clone().to(gpu), 0.5, None), z.double() * 0.5) < 1e-6


# ---------------------------------------------------------------- windowed attention
def run_window(gpu, p, wq, wk, H, G, D, Dv, window, scale, slopes, cuts, eps=1e-3, out_scale=1.0, ring=None, n_splits=None):
    """p [B, T, (H + G) D + G Dv] through qk_norm and window_attention in portions -> [B, T, H * Dv]."""
    B, T, n = p.shape
    ring = ring or ops.WindowRing(B, G, D, Dv, window, p.dtype, gpu)
    outs, at = [], 0
    for L in cuts:
        rows = p[:, at:at + L].reshape(B * L, n).to(gpu)
        step = Step(B, L, at)
        q, k, v = rows[:, :H * D], rows[:, H * D:(H + G) * D], rows[:, (H + G) * D:]
        qn, kn = ops.qk_norm(q, k, v, wq.to(gpu), wk.to(gpu), H, eps, ring, step)
        out = torch.empty(B * L, H * Dv + 8, dtype=p.dtype, device=gpu)[:, 8 * (D % 2 == 0):][:, :H * Dv]
        ops.window_attention(qn, ring, None if slopes is None else slopes.float().to(gpu), scale, step, out, out_scale, kn, None if kn is None else v,
                             n_splits)
        outs.append(out.float().cpu().view(B, L, -1))
        at += L
    return torch.cat(outs, 1)


def window_oracle(p, wq, wk, H, G, D, Dv, window, scale, slopes, eps=1e-3):
    T = p.shape[0]
    p = p.double()
    # (the kernels keep q and k in the dtype)
    q = ko.rms_norm(p[:, :H * D], wq.double(), eps).view(T, H, D)
    k = ko.rms_norm(p[:, H * D:(H + G) * D], wk.double(), eps).view(T, G, D)
    s = torch.zeros(H).double() if slopes is None else slopes.double()
    return ko.window_attention_fast(q, k, p[:, (H + G) * D:].view(T, G, Dv), scale, s, window)


@pytest.mark.parametrize("H,G,D,Dv,window", [(4, 2, 32, 64, 40), (6, 1, 64, 32, 33), (2, 2, 128, 128, 150), (20, 1, 40, 24, 64), (1, 1, 136, 256, 17),
                                             (3, 3, 20, 12, 7), (4, 4, 5, 9, 1), (8, 2, 48, 96, 65), (2, 1, 256, 128, 300)])
def test_window_attention(gpu, H, G, D, Dv, window):
    """Prompts, portions of every path and decoding; scores sharp enough that a key more or less at the window's edge shows."""
    T, B = 330, 2
    g = torch.Generator().manual_seed(H * 1000 + D)
    for dt in ("f32", "bf16", "f16"):
        p = rand(g, B, T, (H + G) * D + G * Dv, dt=dt)
        wq, wk = (1 + rand(g, H * D, s=0.2)).to(DT[dt]), (1 + rand(g, G * D, s=0.2)).to(DT[dt])
        scale, slopes = 1.4 * D ** -0.5, ko.distance_slopes(H)
        want = torch.stack([window_oracle(p[b], wq, wk, H, G, D, Dv, window, scale, slopes) for b in range(B)])
        tol = TOL[dt] if dt == "f32" else 2 * TOL[dt]
        for other in (window - 1, window + 1):
            if 1 < window <= T // 2:
                assert err(window_oracle(p[0], wq, wk, H, G, D, Dv, other, scale, slopes), want[0]) > 2 * tol
        for cuts in ([T], cut(T, [16]), cut(T, [2, 17, 1, 64, 3, 100]), [40] + [1] * (T - 40), cut(T, [33, 5])):
            assert err(run_window(gpu, p, wq, wk, H, G, D, Dv, window, scale, slopes, cuts), want) < tol, (dt, cuts[:6])
        assert err(run_window(gpu, p, wq, wk, H, G, D, Dv, window, scale, None, cut(T, [7, 31]), out_scale=0.5), 0.5 * torch.stack(
            [window_oracle(p[b], wq, wk, H, G, D, Dv, window, scale, None) for b in range(B)])) < tol
        for n in (2, 5, 64):                             # slices, some of them empty
            assert err(run_window(gpu, p, wq, wk, H, G, D, Dv, window, scale, slopes, cut(T, [9]), n_splits=n), want) < tol, (dt, n)


def test_one_key_at_the_windows_edge(gpu):
    """One key stands out; queries just inside and just outside its reach, in prompts and in decoding, at every offset of the
    ring's and the tiles' borders."""
    H, G, D, Dv = 2, 1, 64, 64
    for window in (63, 64, 65, 100):
        for at in (0, 31, 63, 64, 127, 128):
            T = at + window + 3
            g = torch.Generator().manual_seed(at)
            p = rand(g, 1, T, (H + G) * D + G * Dv, dt="bf16", s=0.3)
            p[:, :, :H * D] += 1.0                                  # every query looks the same way,
            p[:, :, H * D:(H + G) * D] *= 0.2
            p[:, at, H * D:(H + G) * D] = 1.0                       # and so does this key
            wq, wk = torch.ones(H * D).bfloat16(), torch.ones(G * D).bfloat16()
            args = (H, G, D, Dv, window, 0.4, torch.tensor([0.01, 0.001]))
            want = window_oracle(p[0], wq, wk, *args)
            last = at + window - 1
            assert float((want[last] - want[last + 1]).abs().max()) > 0.3
            for cuts in ([T], [max(at, 1)] + [1] * (T - max(at, 1)), cut(T, [16]), cut(T, [48])):
                assert err(run_window(gpu, p, wq, wk, *args, cuts), want[None]) < 1.5e-2, (window, at, cuts[:3])


# ---------------------------------------------------------------- gated delta rule
def delta_case(g, B, T, G, H, dim, vdim, taps, dt):
    kd, vd = G * dim, H * vdim
    t = {"p": rand(g, B, T, 2 * kd + vd + H, dt=dt), "a": rand(g, B, T, H * dim, dt=dt, s=2.0), "gate": rand(g, B, T, vd, dt=dt), "A_log": rand(g, H, dt=dt) - 1,
         "dt_bias": rand(g, H * dim, dt=dt), "norm": 1 + rand(g, vdim, dt=dt, s=0.2)}
    for n, c in (("q", kd), ("k", kd), ("v", vd)):
        t["w_" + n] = rand(g, c, taps, dt=dt, s=0.7)
    return t


def delta_oracle(t, b, first, G, H, dim, vdim, eps):
    p, kd, vd = t["p"][b, first:].double(), G * dim, H * vdim
    T = p.shape[0]
    dt = t["p"].dtype
    conv = lambda x, n: ko.silu(ko.causal_conv(x, t["w_" + n].double())).to(dt).double()      # (the kernels keep these in the dtype)
    q = ko.unit(conv(p[:, :kd], "q").view(T, G, dim)) * dim ** -0.5
    k = ko.unit(conv(p[:, kd:2 * kd], "k").view(T, G, dim))
    v = conv(p[:, 2 * kd:2 * kd + vd], "v").view(T, H, vdim)
    beta = torch.sigmoid(p[:, 2 * kd + vd:])
    decay = torch.exp(-torch.exp(t["A_log"].double())[:, None] * ko.softplus(t["a"][b, first:].double() + t["dt_bias"].double()).view(T, H, dim))
    o = ko.delta_rule(q, k, v, decay, beta)
    return o.reshape(T, -1), ko.rms_norm(o, t["norm"].double(), eps).reshape(T, -1) * torch.sigmoid(t["gate"][b, first:].double())


def delta_run(gpu, t, cuts, G, H, dim, vdim, taps, eps, start=None, S=None, conv=None, out_scale=1.0):
    B, T, n = t["p"].shape
    kd, vd = G * dim, H * vdim
    d = {k: v.to(gpu) for k, v in t.items()}
    conv = conv or layer_ops.ConvState(B, taps, 2 * kd + vd, gpu)
    S = torch.zeros(B, H, vdim, dim, device=gpu) if S is None else S
    raw, outs, at = [], [], 0
    for L in cuts:
        step = Step(B, L, at, None, start)
        rows = d["p"][:, at:at + L].reshape(B * L, n)
        x = ops.delta_prep(rows[:, :kd], rows[:, kd:2 * kd], rows[:, 2 * kd:2 * kd + vd], rows[:, 2 * kd + vd:], d["a"][:, at:at + L].reshape(B * L, -1),
                           d["w_q"], d["w_k"], d["w_v"], d["A_log"], d["dt_bias"], conv, dim, vdim, step)
        o = ops.delta_scan(x, S, step)
        out = torch.empty(B * L, vd + 4, dtype=rows.dtype, device=gpu)[:, 4:]
        ops.head_norm_gate(o, d["norm"], d["gate"][:, at:at + L].reshape(B * L, -1), H, eps, out, out_scale)
        raw.append(o.cpu().view(B, L, -1))
        outs.append(out.float().cpu().view(B, L, -1))
        at += L
    return torch.cat(raw, 1), torch.cat(outs, 1), S, conv


@pytest.mark.parametrize("G,H,dim,vdim,taps", [(2, 4, 32, 48, 3), (1, 1, 64, 64, 4), (3, 3, 7, 10, 7), (1, 3, 128, 128, 4), (2, 2, 16, 5, 1), (1, 2, 200, 24, 2),
                                               (2, 2, 64, 128, 5), (1, 1, 256, 256, 16), (4, 4, 128, 64, 4)])
def test_delta_rule(gpu, G, H, dim, vdim, taps):
    B, T, eps = 2, 150, 1e-4
    g = torch.Generator().manual_seed(dim * 7 + taps)
    for dt in ("f32", "bf16", "f16"):
        t = delta_case(g, B, T, G, H, dim, vdim, taps, dt)
        want = [delta_oracle(t, b, 0, G, H, dim, vdim, eps) for b in range(B)]
        w_raw, w_out = torch.stack([w[0] for w in want]), torch.stack([w[1] for w in want])
        for cuts in ([T], cut(T, [1]), cut(T, [2]), cut(T, [32, 33, 1]), [65, 64, 21], cut(T, [17, 16, 3])):
            raw, out, _, _ = delta_run(gpu, t, cuts, G, H, dim, vdim, taps, eps)
            assert err(raw, w_raw) < (2e-5 if dt == "f32" else TOL[dt]) and err(out, w_out) < (5e-5 if dt == "f32" else 2 * TOL[dt]), (dt, cuts[:4])
        start = torch.tensor([0, 41], dtype=torch.int32, device=gpu)          # left padding
        t["p"][1, :41], t["a"][1, :41] = 7.0, 7.0
        raw, out, _, _ = delta_run(gpu, t, cut(T, [29, 31]), G, H, dim, vdim, taps, eps, start)
        w_raw, w_out = delta_oracle(t, 1, 41, G, H, dim, vdim, eps)
        assert err(raw[1, 41:], w_raw) < (2e-5 if dt == "f32" else TOL[dt]) and bool((raw[1, :41] == 0).all())


def test_delta_rule_remembers_and_overwrites(gpu):
    """Slow decays: the first token's value is read back hundreds of tokens later, unless its key is written again."""
    dim, vdim, T = 64, 32, 400
    g = torch.Generator().manual_seed(5)
    for dt in ("f32", "bf16"):
        t = delta_case(g, 1, T, 1, 1, dim, vdim, 2, dt)
        t["A_log"].fill_(-9.0)
        for n in ("w_q", "w_k", "w_v"):
            t[n].zero_()
            t[n][:, -1] = 1.0
        p = t["p"]
        p[:, :, :2 * dim] = -8.0                                    # (silu of it is nearly nothing)
        basis = torch.arange(T) % (dim // 2)
        for i in range(T):
            p[0, i, dim + 1 + basis[i] % (dim // 2 - 1)] = 4.0      # keys that never meet channel 0 ...
        p[0, 0, dim:2 * dim] = -8.0
        p[0, 0, dim] = 4.0                                          # ... which the first token writes
        p[0, 350, dim:2 * dim] = -8.0
        p[0, 350, dim] = 4.0                                        # and this one writes again
        p[0, 300:, :dim] = -8.0
        p[0, 300:, 0] = 4.0                                         # queries for it
        p[:, :, -1] = 6.0
        want = delta_oracle(t, 0, 0, 1, 1, dim, vdim, 1e-4)[0]
        assert float((want[349] - want[351]).abs().max()) > 0.1 * float(want.abs().max())
        for cuts in ([T], [290] + [1] * 110, cut(T, [64]), cut(T, [50, 3])):
            assert err(delta_run(gpu, t, cuts, 1, 1, dim, vdim, 2, 1e-4)[0], want[None]) < TOL[dt], (dt, cuts[:3])


def test_delta_rule_with_decays_that_vanish(gpu):
    """Decays from none at all to exp(-200) within a token, mixed over channels and time."""
    G, H, dim, vdim, T = 1, 2, 128, 64, 300
    g = torch.Generator().manual_seed(6)
    for dt in ("f32", "bf16"):
        t = delta_case(g, 1, T, G, H, dim, vdim, 4, dt)
        t["A_log"] = torch.tensor([4.0, -2.0]).to(DT[dt])
        t["a"] = (t["a"].float() * 4).to(DT[dt])
        want = delta_oracle(t, 0, 0, G, H, dim, vdim, 1e-4)[0]
        for cuts in ([T], cut(T, [100, 1, 65])):
            assert err(delta_run(gpu, t, cuts, G, H, dim, vdim, 4, 1e-4)[0], want[None]) < TOL[dt], (dt, cuts[:3])


# ---------------------------------------------------------------- matrix memory
def memory_run(gpu, p, b_i, b_f, w, H, dim, vdim, cap, eps, cuts, start=None, state=None):
    B, T, n = p.shape
    S, m = state or ops.memory_state(B, H, dim, vdim, gpu)
    o1, o2, o3 = H * dim, 2 * H * dim, 2 * H * dim + H * vdim
    raw, outs, at = [], [], 0
    for L in cuts:
        step = Step(B, L, at, None, start)
        r = p[:, at:at + L].reshape(B * L, n).to(gpu)
        li, lf = ops.memory_gates(r[:, -2 * H:-H], r[:, -H:], b_i.to(gpu), b_f.to(gpu), cap)
        o, den = ops.memory_scan(r[:, :o1], r[:, o1:o2], r[:, o2:o3], li, lf, S, m, dim ** -0.5, step)
        out = torch.empty(B * L, H * vdim, dtype=p.dtype, device=gpu)
        ops.head_norm_gate(o, w.to(gpu), r[:, o3:o3 + H * vdim], H, eps, out, 1.0, den)
        raw.append((o.view(B, L, H, vdim) / den.view(B, L, H, 1)).cpu().view(B, L, -1))
        outs.append(out.float().cpu().view(B, L, -1))
        at += L
    return torch.cat(raw, 1), torch.cat(outs, 1)


def memory_oracle(p, b_i, b_f, w, H, dim, vdim, cap, eps):
    T = p.shape[0]
    p = p.double()
    o1, o2, o3 = H * dim, 2 * H * dim, 2 * H * dim + H * vdim
    li = ko.cap(p[:, -2 * H:-H] + b_i.double(), cap)
    lf = ko.log_sigmoid(ko.cap(p[:, -H:] + b_f.double(), cap))
    o = ko.matrix_memory(p[:, :o1].view(T, H, dim) * dim ** -0.5, p[:, o1:o2].view(T, H, dim), p[:, o2:o3].view(T, H, vdim), li, lf)
    return o.reshape(T, -1), ko.rms_norm(o, None, eps).reshape(T, -1) * w.double() * torch.sigmoid(p[:, o3:o3 + H * vdim])


@pytest.mark.parametrize("H,dim,vdim,cap", [(3, 16, 40, 7.0), (1, 64, 64, 15.0), (5, 9, 6, 4.0), (2, 128, 128, 12.0), (2, 200, 24, 9.0), (1, 256, 300, 5.0), (4, 32, 64, 30.0)])
def test_matrix_memory(gpu, H, dim, vdim, cap):
    B, T, eps = 2, 170, 1e-4
    g = torch.Generator().manual_seed(dim + H)
    for dt in ("f32", "bf16", "f16"):
        p = rand(g, B, T, 2 * H * dim + 2 * H * vdim + 2 * H, dt=dt)
        p[:, :, -2 * H:-H] *= 3.0                                # input gates that move the running maximum about
        b_i, b_f, w = rand(g, H, dt=dt), 3 + rand(g, H, dt=dt), (1 + rand(g, H * vdim, s=0.2)).to(DT[dt])
        want = [memory_oracle(p[b], b_i, b_f, w, H, dim, vdim, cap, eps) for b in range(B)]
        w_raw, w_out = torch.stack([x[0] for x in want]), torch.stack([x[1] for x in want])
        for cuts in ([T], cut(T, [1]), cut(T, [2]), cut(T, [64, 65, 1]), cut(T, [17, 16, 3])):
            raw, out = memory_run(gpu, p, b_i, b_f, w, H, dim, vdim, cap, eps, cuts)
            # (a normalizer near zero magnifies rounding: judged where it does not)
            assert err(out, w_out) < (1e-4 if dt == "f32" else 2.5 * TOL[dt]), (dt, cuts[:4])
            assert float(((raw.double() - w_raw).pow(2).mean() / w_raw.pow(2).mean()).sqrt()) < (1e-3 if dt == "f32" else 0.1), (dt, cuts[:4])
        start = torch.tensor([0, 41], dtype=torch.int32, device=gpu)          # left padding
        p[1, :41] = 7.0
        _, out = memory_run(gpu, p, b_i, b_f, w, H, dim, vdim, cap, eps, cut(T, [29, 31]), start)
        assert err(out[1, 41:], memory_oracle(p[1, 41:], b_i, b_f, w, H, dim, vdim, cap, eps)[1]) < (1e-4 if dt == "f32" else 2.5 * TOL[dt])


def test_matrix_memory_recalls_a_far_token(gpu):
    """One token with a large input gate among hundreds with small ones."""
    H, dim, vdim, T, cap = 1, 64, 48, 500, 12.0
    g = torch.Generator().manual_seed(9)
    for dt in ("f32", "bf16"):
        p = rand(g, 1, T, 2 * H * dim + 2 * H * vdim + 2 * H, dt=dt)
        p[:, :, -2] = -6.0
        p[:, :, -1] = 40.0
        for far in (0, 63, 64, 130):
            q = p.clone()
            q[:, far, -2] = 10.0
            b, w = torch.zeros(1).to(DT[dt]), torch.ones(vdim).to(DT[dt])
            want = memory_oracle(q[0], b, b, w, H, dim, vdim, cap, 1e-4)[1]
            assert err(memory_oracle(p[0], b, b, w, H, dim, vdim, cap, 1e-4)[1][-50:], want[-50:]) > 0.3
            for cuts in ([T], [440] + [1] * 60, cut(T, [100, 2])):
                assert err(memory_run(gpu, q, b, b, w, H, dim, vdim, cap, 1e-4, cuts)[1], want[None]) < (2e-4 if dt == "f32" else 2.5 * TOL[dt]), (dt, far)


# ---------------------------------------------------------------- chunked recurrences, longer calls
@pytest.mark.parametrize("workspace", [1, 400_000, 3_000_000, 384 << 20])
def test_chunks_in_segments(gpu, monkeypatch, workspace):
    """Workspaces of one chunk, of a few, and of the whole call, whose segments are then made on a second stream while others
    are walked; state handed from segment to segment and from call to call, the last chunk partial."""
    monkeypatch.setattr(ops, "WORKSPACE_BYTES", workspace)
    g = torch.Generator().manual_seed(11)
    T = 4500
    for cuts in ([T], [4200, 1, 299]):
        t = delta_case(g, 1, T, 1, 2, 48, 20, 3, "bf16")
        t["A_log"] -= 3.0                                        # (memories of hundreds of tokens)
        want = delta_oracle(t, 0, 0, 1, 2, 48, 20, 1e-4)[0]
        assert err(delta_run(gpu, t, cuts, 1, 2, 48, 20, 3, 1e-4)[0], want[None]) < TOL["bf16"], cuts
        p = rand(g, 1, T, 2 * 32 + 2 * 20 + 2, dt="bf16")
        p[:, :, -1] += 5.0
        b, w = torch.zeros(1).bfloat16(), torch.ones(20).bfloat16()
        want = memory_oracle(p[0], b, b, w, 1, 32, 20, 9.0, 1e-4)[1]
        assert err(memory_run(gpu, p, b, b, w, 1, 32, 20, 9.0, 1e-4, cuts)[1], want[None]) < 2.5 * TOL["bf16"], cuts


def test_chunks_agree_with_the_token_by_token_kernel(gpu, monkeypatch):
    """A batch of many heads, whose results the plain implementation would take too long for."""
    g = torch.Generator().manual_seed(12)
    B, T, G, H, dim, vdim = 3, 700, 4, 8, 128, 128
    t = delta_case(g, B, T, G, H, dim, vdim, 4, "bf16")
    p = rand(g, B, T, 2 * H * 128 + 2 * H * 192 + 2 * H, dt="bf16")
    p[:, :, -H:] += 4.0
    b, w = torch.zeros(H).bfloat16(), torch.ones(H * 192).bfloat16()
    start = torch.tensor([0, 333, 699], dtype=torch.int32, device=gpu)
    runs = []
    for tokens in (10 ** 9, 1):
        monkeypatch.setattr(ops, "CHUNKED_TOKENS", tokens)
        runs.append((delta_run(gpu, t, [T], G, H, dim, vdim, 4, 1e-4, start), memory_run(gpu, p, b, b, w, H, 128, 192, 12.0, 1e-4, [T], start)))
    (d0, m0), (d1, m1) = runs
    assert err(d1[0], d0[0].double()) < 1e-4 and err(d1[2], d0[2].double().cpu()) < 1e-4 and torch.equal(d1[3].rows, d0[3].rows)
    first = start.tolist()
    for i in range(B):
        assert err(m1[1][i, first[i]:], m0[1][i, first[i]:].double()) < 1e-2


def test_chunks_in_a_graph(gpu):
    """Both streams of a long call captured; several replays with the program's own work between them, each from the same state."""
    g = torch.Generator().manual_seed(13)
    T, H, dim, vdim = 4200, 2, 64, 32
    x = ops.DeltaInputs(*[rand(g, T, n, dt="bf16").to(gpu) for n in (H * dim, H * dim, H * vdim)], torch.full((T, H), 0.01, device=gpu),
                        torch.full((T, H), 0.1, device=gpu), -rand(g, T, H * dim).abs().to(gpu) * 0.02, torch.rand(T, H, generator=g).to(gpu))
    S = torch.zeros(1, H, vdim, dim, device=gpu)
    step = Step(1, T, 0)
    want = ops.delta_scan(x, S, step).clone()
    end = S.clone()
    side = torch.cuda.Stream()
    side.wait_stream(torch.cuda.current_stream())
    with torch.cuda.stream(side):
        S.zero_()
        ops.delta_scan(x, S, step)
    torch.cuda.current_stream().wait_stream(side)
    graph = torch.cuda.CUDAGraph()
    with torch.cuda.graph(graph):
        got = ops.delta_scan(x, S, step)
    for _ in range(4):
        S.zero_()
        graph.replay()
        assert torch.equal(got, want) and torch.equal(S, end)
        torch.cuda.synchronize()
        _ = (got * 2).sum().item()
