"""The Kapudra oracle against library routines and closed forms, configuration, registry and checkpoint handling, the order of
layer runs, and the argument checks of its C ABI.  No GPU."""
import json
import math

import pytest
import torch
import torch.nn.functional as F

from oracle import kapudra_oracle as ko
from polarquant_amd import _ffi
from polarquant_amd import build as pq_build
from polarquant_amd import checkpoint as ck
from polarquant_amd.modeling_kapudra import KapudraConfig, KapudraForCausalLM
from polarquant_amd.modeling_recurrent import Loop, Packed, distance_slopes, layer_runs
from polarquant_amd.registry import family_of

import kapudra_cases as kc


# ---------------------------------------------------------------- oracle
def test_oracle_elementwise_against_library_routines():
    x = torch.linspace(-30, 30, 401).double()
    assert torch.allclose(ko.gelu_tanh(x), F.gelu(x, approximate="tanh"), atol=1e-12)
    assert torch.allclose(ko.silu(x), F.silu(x), atol=1e-12) and torch.allclose(ko.softplus(x), F.softplus(x, threshold=1000), atol=1e-12)
    assert torch.allclose(ko.log_sigmoid(x), F.logsigmoid(x), atol=1e-12)
    assert torch.allclose(ko.rms_norm(x.view(1, -1), None, 1e-3), F.rms_norm(x.view(1, -1), (401,), None, 1e-3), atol=1e-12)
    w = torch.randn(6, 4, generator=torch.Generator().manual_seed(0)).double()
    s = torch.randn(9, 6, generator=torch.Generator().manual_seed(1)).double()
    assert torch.allclose(ko.causal_conv(s, w), F.conv1d(F.pad(s.T[None], (3, 0)), w[:, None], groups=6)[0].T, atol=1e-12)


def test_oracle_attention_against_library_softmax():
    g = torch.Generator().manual_seed(1)
    q, k, v = torch.randn(11, 4, 8, generator=g).double(), torch.randn(11, 2, 8, generator=g).double(), torch.randn(11, 2, 6, generator=g).double()
    slopes = ko.distance_slopes(4)
    assert torch.allclose(slopes, torch.tensor([0.25, 1 / 16, 1 / 64, 1 / 256]).double()) and torch.equal(distance_slopes(4).double(), slopes)
    for window in (1, 3, 11, None):
        got = ko.window_attention(q, k, v, 0.4, slopes, window)
        assert torch.allclose(got, ko.window_attention_fast(q, k, v, 0.4, slopes, window), atol=1e-12)
        back = torch.arange(11)[:, None] - torch.arange(11)[None, :]
        bias = -slopes[:, None, None] * back + torch.where((back >= 0) & (back < (window or 99)), 0.0, -math.inf)
        rep = lambda t: t.repeat_interleave(2, 1).transpose(0, 1)[None]
        want = F.scaled_dot_product_attention(q.transpose(0, 1)[None], rep(k), rep(v), attn_mask=bias[None], scale=0.4)
        assert torch.allclose(got, want[0].transpose(0, 1).reshape(11, -1), atol=1e-9)


def test_oracle_recurrences_against_closed_forms():
    g = torch.Generator().manual_seed(2)
    T, d, dv = 7, 5, 4
    q, k, v = [torch.randn(T, 1, n, generator=g).double() for n in (d, d, dv)]
    # without decay a full step overwrites what the unit key holds
    ku = ko.unit(k)
    one = torch.ones(T, 1).double()
    o = ko.delta_rule(ku, ku, v, torch.ones(T, 1, d).double(), one)
    assert torch.allclose(o, v, atol=1e-5)
    # without steps, or forgetting all, only the newest token remains
    beta = torch.rand(T, 1, generator=g).double()
    last = ko.delta_rule(q, ku, v, torch.zeros(T, 1, d).double(), beta)
    assert torch.allclose(last, (q * ku).sum(-1, keepdim=True) * beta[..., None] * v, atol=1e-12)
    # a matrix memory is a normalized weighted sum
    li, lf = torch.randn(T, 1, generator=g).double(), F.logsigmoid(torch.randn(T, 1, generator=g).double())
    o = ko.matrix_memory(q, k, v, li, lf)
    for t in range(T):
        w = torch.stack([li[s, 0] + lf[s + 1:t + 1, 0].sum() for s in range(t + 1)])
        m = max(float(lf[:t + 1].sum()), float(w.max()))
        # (the running maximum begins at 0 and takes part)
        m = 0.0
        for s in range(t + 1):
            m = max(float(lf[s]) + m, float(li[s]))
        p = torch.exp(w - m) * (k[:t + 1, 0] @ q[t, 0])
        assert torch.allclose(o[t, 0], (p @ v[:t + 1, 0]) / (max(abs(float(p.sum())), math.exp(-m)) + 1e-6), atol=1e-10)


def test_oracle_slow_and_fast_forward_agree():
    w = kc.weights(kc.ODD, 3)
    t = kc.tokens(11, kc.ODD["vocab"], 4)
    assert torch.allclose(ko.forward(t, kc.ODD, w), ko.forward(t, kc.ODD, w, slow=True), atol=1e-10)


def test_every_mechanism_shows():
    """Changing a constant or a tensor changes the logits by more than the tolerance of the comparisons on the GPU (1e-4), so that
    they would notice it."""
    cfg = kc.changed(kc.EVEN, lambda c: (c.update(logit_softcap=2.0), [c["layers"][i]["mixer"]["left"].update(scale=1.0) for i in (0, 2)]))   # (sharp attention)
    w = kc.weights(cfg, 13, kc.RANKS["even"])
    t = kc.tokens(56, cfg["vocab"], 6)
    want = ko.forward(t, cfg, w)
    off = lambda c=cfg, x=w: kc.rel_rms(ko.forward(t, c, x), want)
    left = lambda c, i: c["layers"][i]["mixer"]["left"]
    for change in (lambda c: left(c, 0)["mask"].update(size=39), lambda c: left(c, 0)["mask"].update(size=41), lambda c: left(c, 2).update(scale=1.05),
                   lambda c: c["layers"][0]["mixer"].update(left_scale=0.51), lambda c: c["layers"][0]["mixer"].update(right_scale=1.21),
                   lambda c: c["layers"][1]["mixer"].update(gate_cap=7.5), lambda c: c.update(logit_scale=0.71), lambda c: c.update(logit_softcap=2.2),
                   lambda c: c["embedding"].update(scale=3.1), lambda c: c["loop"].update(times=2), lambda c: c["norm"].update(eps=1e-3)):
        assert off(kc.changed(cfg, change)) > 5e-4
    g = torch.Generator().manual_seed(1)
    for name, v in w.items():
        if name.startswith("l2.") or name.startswith("l3."):         # (kinds of tensors that the first two layers have)
            continue
        r = torch.randn(v.shape, generator=g)
        assert off(x=dict(w, **{name: v + 4.0 * r if name.endswith(".b") and v.dim() == 1 else v * (1 + 0.5 * r)})) > 5e-4, name


# ---------------------------------------------------------------- configuration, registry, checkpoint
def test_config_round_trip_and_registry():
    for cfg in kc.ALL.values():
        c = KapudraConfig.from_dict(cfg)
        assert c.to_dict() == cfg and KapudraConfig.from_dict(json.loads(json.dumps(c.to_dict()))) == c
    fam = family_of(kc.EVEN)
    assert fam.model_class() is KapudraForCausalLM and not fam.polar_cache and fam.libraries == ("steps", "recurrent")
    assert set(fam.libraries) <= set(pq_build.LAYER_LIBS)


@pytest.mark.parametrize("change,message", [
    (lambda c: c["layers"][0].update(type="other"), "mixer type"),
    (lambda c: c["layers"][0]["mlp"].update(kind="experts"), "kind"),
    (lambda c: c["layers"][0]["mixer"]["left"].update(rope=7), "not implemented"),
    (lambda c: c["layers"][0]["mixer"]["left"]["mask"].update(sinks=7), "not implemented"),
    (lambda c: c["layers"][1]["mixer"].update(conv=4), "not implemented"),
    (lambda c: c["loop"].update(stop=9), "no loop"),
    (lambda c: c["loop"].update(times=0), "no loop"),
])
def test_config_refuses_what_is_not_implemented(change, message):
    with pytest.raises(ValueError, match=message):
        KapudraConfig.from_dict(kc.changed(kc.EVEN, change))


def test_order_of_layer_runs():
    assert layer_runs(4, Loop(1, 3, 2)) == [(0, None), (1, 0), (2, None), (1, 1), (2, None), (3, None)]
    assert layer_runs(2, None) == [(0, None), (1, None)] and layer_runs(1, Loop(0, 1, 3)) == [(0, 0), (0, 1), (0, 2)]
    for cfg in kc.ALL.values():
        assert layer_runs(len(cfg["layers"]), KapudraConfig.from_dict(cfg).loop) == ko.schedule(cfg)


@pytest.mark.parametrize("name", sorted(kc.ALL))
def test_checkpoint_directory(tmp_path, name):
    cfg = kc.ALL[name]
    w = kc.write(str(tmp_path / "a"), cfg, 5, kc.RANKS[name])
    model = ck.load_pretrained(str(tmp_path / "a"), torch.bfloat16, "cpu", cache_capacity=77)
    assert isinstance(model, KapudraForCausalLM)
    for _ in range(2):                                      # before and after the projections are packed
        got = model.checkpoint_tensors()
        assert set(got) == set(w) and all(torch.equal(got[n], w[n]) for n in w)
        assert len(list(model.parameters())) == len(w)
        for layer in model.model.layers:
            rows = layer._in.weight()
            assert rows.shape[0] % 16 == 0 and layer._out.weight().shape[1] % 32 == 0
            assert layer._in.weight().data_ptr() == rows.data_ptr()
    ck.save_pretrained(model, str(tmp_path / "b"), shards=2)
    again = ck.load_pretrained(str(tmp_path / "b"), torch.float32, "cpu").checkpoint_tensors()
    assert all(torch.equal(again[n], w[n].float()) for n in w)
    with open(tmp_path / "b" / "config.json") as f:
        assert json.load(f) == cfg
    with pytest.raises(TypeError):
        ck.load_pretrained(str(tmp_path / "a"), torch.bfloat16, "cpu", rbits=4)       # not a polar-key model
    assert model.kv_cache_bytes_per_token() == 0 and model.state_bytes() > 0


def test_checkpoint_must_hold_every_tensor(tmp_path):
    w = kc.weights(kc.EVEN, 1)
    for gone in ("l0.mix.right.a1", "l1.mix.f.b", "loop.step"):
        kc.write(str(tmp_path / gone), kc.EVEN, 0, w={k: v for k, v in w.items() if k != gone})
        with pytest.raises(KeyError, match=gone):
            ck.load_pretrained(str(tmp_path / gone), torch.bfloat16, "cpu")


def test_packed_parameters_are_slices_and_follow_a_move():
    a, b = torch.nn.Parameter(torch.randn(3, 4)), torch.nn.Parameter(torch.randn(5, 4))
    va, vb = a.detach().clone(), b.detach().clone()
    p = Packed([(a, 8), (b, 8)], 0, 32)
    w = p.weight()
    assert w.shape == (32, 4) and torch.equal(w[:3], va) and torch.equal(w[8:13], vb) and float(w[3:8].abs().sum() + w[13:].abs().sum()) == 0
    with torch.no_grad():
        b.zero_()
    assert float(p.weight()[8:13].abs().sum()) == 0 and p.weight().data_ptr() == w.data_ptr()
    b.data = vb.double().float().clone()
    assert torch.equal(p.weight()[8:13], vb)
    c = Packed([(torch.nn.Parameter(va), 8), (torch.nn.Parameter(va * 2), 8)], 1, 32)
    assert c.weight().shape == (3, 32) and torch.equal(c.weight()[:, 8:12], va * 2)


# ---------------------------------------------------------------- C ABI argument checks
A = 0x1000                    # a stand-in address; nothing is launched by the validators
OK, NUL, SHAPE, DTYPE, ALIGN, STRIDE, WS = 0, -1, -2, -4, -5, -6, -7


def test_window_arguments_and_plan():
    lib = _ffi.recurrent_lib()

    def call(**kw):
        d = dict(q=A, kr=A, vr=A, kn=None, ks=0, vn=None, vs=0, sl=A, start=None, pd=None, pos=100, out=A, os=64, B=2, L=3, H=4, G=2, D=24, Dv=16, cap=64,
                 w=49, S=1, ws=None, n=0, dt=1)
        d.update(kw)
        return lib.pq_validate_window_attn(*[d[k] for k in ("q", "kr", "vr", "kn", "ks", "vn", "vs", "sl", "start", "pd", "pos", "out", "os", "B", "L", "H", "G",
                                                            "D", "Dv", "cap", "w", "S", "ws", "n", "dt")])
    assert call() == OK and call(sl=None) == OK and call(dt=2) == OK
    assert call(w=50) == SHAPE and call(w=0) == SHAPE and call(cap=96) == SHAPE and call(H=5) == SHAPE and call(L=17) == SHAPE and call(pos=-1) == SHAPE
    assert call(kn=A) == NUL and call(q=None) == NUL and call(dt=4) == DTYPE and call(os=63) == STRIDE and call(q=A + 1) == ALIGN
    new = dict(kn=A, ks=48, vn=A, vs=32)
    assert call(L=200, **new) == OK and call(L=200, **dict(new, ks=47)) == STRIDE and call(pd=A, **new) == SHAPE
    need = lib.pq_window_workspace_bytes(2, 3, 4, 16, 3)
    assert need == (2 * 3 * 4 * 3 * 2 + 2 * 3 * 4 * 3 * 16) * 4 and lib.pq_window_workspace_bytes(2, 3, 4, 16, 1) == 0
    assert call(S=3, ws=A, n=need) == OK and call(S=3, ws=A, n=need - 1) == WS and call(S=3) == WS and call(S=0) == WS and call(S=65) == WS
    for args in ((1, 1, 32, 8, 4096), (8, 1, 32, 8, 1024), (4096, 1, 1, 1, 5), (1, 16, 64, 1, 10 ** 6)):
        assert 1 <= lib.pq_window_plan(*args, 256) <= 64


def test_delta_arguments():
    lib = _ffi.recurrent_lib()

    def call(**kw):
        d = dict(B=1, L=40, G=2, H=4, dim=16, vdim=24, taps=4, si=A, so=2 * A, rs=96, ars=64, dt=0)
        d.update(kw)
        return lib.pq_validate_delta_prep(*d.values())
    assert call() == OK and call(taps=1, si=None, so=None) == OK and call(L=32, so=A) == OK
    assert call(so=A) == STRIDE and call(si=None) == NUL and call(taps=17) == SHAPE and call(dim=257) == SHAPE and call(H=3) == SHAPE
    assert call(rs=95) == STRIDE and call(ars=63) == STRIDE and call(dt=3) == DTYPE


def test_ops_refuse_cpu_tensors():
    from polarquant_amd import layer_ops, recurrent_ops
    with pytest.raises(RuntimeError, match="no CPU fallback"):
        layer_ops.gelu_mul(torch.zeros(2, 8), torch.zeros(2, 8))
    with pytest.raises(RuntimeError, match="no CPU fallback"):
        recurrent_ops.memory_gates(torch.zeros(2, 1), torch.zeros(2, 1), torch.zeros(1), torch.zeros(1), 3.0)
