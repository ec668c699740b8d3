"""The Dekipel oracle against library routines, configuration, registry and checkpoint handling, and the argument checks
of the latent-attention C ABI.  No GPU."""
import copy
import json

import pytest
import torch
import torch.nn.functional as F

from oracle import dekipel_oracle as do
from polarquant_amd import _ffi
from polarquant_amd import checkpoint as ck
from polarquant_amd.modeling_dekipel import DekipelConfig, DekipelForCausalLM
from polarquant_amd.modeling_latent import LatentModel
from polarquant_amd.registry import family_of

import dekipel_cases as dc


# ---------------------------------------------------------------- oracle
def test_oracle_norms_and_conv_against_library_routines():
    g = torch.Generator().manual_seed(0)
    x, w = torch.randn(5, 24, generator=g).double(), torch.randn(24, generator=g).double()
    assert torch.allclose(do.rms_norm(x, w, 1e-3), F.rms_norm(x, (24,), w, 1e-3), atol=1e-12)
    parts = torch.cat([F.rms_norm(x[:, i * 8:(i + 1) * 8], (8,), None, 1e-3) for i in range(3)], -1) * w
    assert torch.allclose(do.grouped_rms_norm(x, w, 1e-3, 3), parts, atol=1e-12)
    assert not torch.allclose(do.grouped_rms_norm(x, w, 1e-3, 3), do.grouped_rms_norm(x, w, 1e-3, 1), atol=1e-2)
    cw = torch.randn(24, 4, generator=g).double()
    want = x + F.conv1d(F.pad(x.T[None], (3, 0)), cw[:, None], groups=24)[0].T
    assert torch.allclose(do.input_conv(x, cw), want, atol=1e-12)


def test_oracle_attention_against_library_softmax():
    g = torch.Generator().manual_seed(1)
    q, k, v = [torch.randn(9, 3, 8, generator=g).double() for _ in range(3)]
    sink = torch.tensor([-1e9, 0.7, 3.0]).double()
    got = do.attend(q, k, v, sink, 0.3)
    assert torch.allclose(got, do.attend_fast(q, k, v, sink, 0.3), atol=1e-12)
    # a sink is a key whose score is the sink itself and whose value is zero
    s = torch.einsum("ihd,jhd->hij", q, k) * 0.3
    s = s.masked_fill(torch.ones(9, 9).triu(1).bool(), -float("inf"))
    p = torch.softmax(torch.cat([s, sink[:, None, None].expand(3, 9, 1)], -1), -1)[..., :-1]
    assert torch.allclose(got, torch.einsum("hij,jhd->ihd", p, v).reshape(9, -1), atol=1e-12)
    assert torch.allclose(got[:, :8], F.scaled_dot_product_attention(*[t[:, :1].transpose(0, 1)[None] for t in (q, k, v)], is_causal=True, scale=0.3)[0, 0], atol=1e-9)


def test_oracle_slow_and_fast_forward_agree():
    w = do.random_weights(dc.ODD, 3)
    t = dc.tokens(11, dc.ODD["vocab"], 4)
    assert torch.allclose(do.forward(t, dc.ODD, w), do.forward(t, dc.ODD, w, slow=True), atol=1e-10)


# ---------------------------------------------------------------- configuration, registry, checkpoint
def test_config_round_trip_and_registry():
    for cfg in dc.ALL.values():
        c = DekipelConfig.from_dict(cfg)
        assert c.to_dict() == cfg and DekipelConfig.from_dict(json.loads(json.dumps(c.to_dict()))) == c
    fam = family_of(dc.EVEN)
    assert fam.model_class() is DekipelForCausalLM and not fam.polar_cache and fam.libraries == ("steps", "latent")
    assert family_of({"model_type": "qwen2"}).name == "qwen2" and family_of({}).name == "llama"
    with pytest.raises(ValueError, match="not one of"):
        family_of({"architecture": "nobody"})


@pytest.mark.parametrize("change,message", [
    (lambda c: c["layers"][0].update(type="other"), "mixer type"),
    (lambda c: c["layers"][0]["mlp"].update(kind="experts"), "kind"),
    (lambda c: c["layers"][0]["mixer"].update(window=7), "not implemented"),
    (lambda c: c["layers"][2]["mixer"].update(kv_from=2), "takes its latents"),
    (lambda c: c["layers"][3]["mixer"].update(kv_from=2), "takes its latents"),       # layer 2 has none of its own
    (lambda c: c["layers"][2]["mixer"].update(kv_from=1), "takes its latents"),       # another rank
])
def test_config_refuses_what_is_not_implemented(change, message):
    c = copy.deepcopy(dc.EVEN)
    change(c)
    with pytest.raises(ValueError, match=message):
        DekipelConfig.from_dict(c)


@pytest.mark.parametrize("name", sorted(dc.ALL))
def test_checkpoint_directory(tmp_path, name):
    cfg = dc.ALL[name]
    w = dc.write(str(tmp_path / "a"), cfg, 5)
    model = ck.load_pretrained(str(tmp_path / "a"), torch.bfloat16, "cpu", cache_capacity=77)
    assert isinstance(model, DekipelForCausalLM) and model.config.cache_capacity == 77
    got = model.checkpoint_tensors()
    assert set(got) == set(w) and all(torch.equal(got[n], w[n]) for n in w)
    assert len(list(model.parameters())) == len(w)
    ck.save_pretrained(model, str(tmp_path / "b"), shards=2)
    again = ck.load_pretrained(str(tmp_path / "b"), torch.float32, "cpu").checkpoint_tensors()
    assert all(torch.equal(again[n], w[n].float()) for n in w)
    with open(tmp_path / "b" / "config.json") as f:
        assert json.load(f) == cfg
    with pytest.raises(TypeError):
        ck.load_pretrained(str(tmp_path / "a"), torch.bfloat16, "cpu", rbits=4)       # not a polar-key model
    own = sum(l["mixer"]["kv_rank"] for l in cfg["layers"] if "kv_from" not in l["mixer"])
    assert model.kv_cache_bytes_per_token() == 2 * own


def test_checkpoint_must_hold_every_tensor(tmp_path):
    w = do.random_weights(dc.PADDED, 1)
    missing = {k: v for k, v in w.items() if k != "l1.mix.sink"}
    dc.write(str(tmp_path / "a"), dc.PADDED, 0, weights=missing)
    with pytest.raises(KeyError, match="l1.mix.sink"):
        ck.load_pretrained(str(tmp_path / "a"), torch.bfloat16, "cpu")
    dc.write(str(tmp_path / "b"), dc.PADDED, 0, weights=dict(w, extra=torch.zeros(2)))
    with pytest.raises(KeyError, match="extra"):
        ck.load_pretrained(str(tmp_path / "b"), torch.bfloat16, "cpu")


def test_a_layer_without_feed_forward_ignores_its_norms(tmp_path):
    w = do.random_weights(dc.EVEN, 2)
    dc.write(str(tmp_path), dc.EVEN, 0, weights=dict(w, **{"l1.norm2": torch.ones(192), "l1.canon2": torch.ones(192, 3)}))
    assert "l1.norm2" not in ck.load_pretrained(str(tmp_path), torch.bfloat16, "cpu").checkpoint_tensors()


def test_left_padding_of_a_mask():
    pad = LatentModel._left_padding
    assert pad(None) is None and pad(torch.ones(2, 5)) is None
    assert pad(torch.tensor([[0, 0, 1, 1], [1, 1, 1, 1]])).tolist() == [2, 0]
    with pytest.raises(ValueError, match="left padding"):
        pad(torch.tensor([[1, 0, 1]]))


# ---------------------------------------------------------------- C ABI argument checks
@pytest.fixture(scope="module")
def lib():
    class Both:                 # the steps' and the latent kernels' symbols
        def __getattr__(self, name):
            return getattr(_ffi.steps_lib() if name in _ffi.STEPS_SIGNATURES else _ffi.latent_lib(), name)
    return Both()


def test_header_and_signatures_name_the_same_symbols(lib):
    import os
    import re
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    seen = set(_ffi.SIGNATURES)
    for header, table, load in (("steps", _ffi.STEPS_SIGNATURES, _ffi.steps_lib), ("latent", _ffi.LATENT_SIGNATURES, _ffi.latent_lib),
                                ("recurrent", _ffi.RECURRENT_SIGNATURES, _ffi.recurrent_lib)):
        with open(os.path.join(root, "include", "polarquant_%s.h" % header)) as f:
            text = re.sub(r"/\*.*?\*/", "", f.read(), flags=re.S)
        found = re.findall(r"\b(pq_\w+)\s*\(([^)]*)\)\s*;", text)
        assert {n for n, _ in found} == set(table) and not seen & set(table)
        for n, args in found:
            assert len(args.split(",")) == len(table[n][1]), n
        seen |= set(table)
        load()


A, B16 = 0x1000, 0x2000       # stand-in addresses; nothing is launched by the validators
OK, NUL, SHAPE, DTYPE, ALIGN, STRIDE, WS = 0, -1, -2, -4, -5, -6, -7


def test_norm_conv_arguments(lib):
    def call(**kw):
        d = dict(x=A, y=B16, wp=A, xo=B16, w=A, cw=A, si=A, so=B16, h=A, start=None, pd=None, pos=0, B=2, L=40, W=64, g=2, taps=4, dt=1)
        d.update(kw)
        return lib.pq_validate_norm_conv(*[d[k] for k in ("x", "y", "wp", "xo", "w", "cw", "si", "so", "h", "start", "pd", "pos", "B", "L", "W", "g", "taps", "dt")])
    assert call() == OK and call(dt=2) == OK and call(L=1, xo=A, so=A) == OK and call(cw=None, si=None, so=None, xo=A) == OK
    assert call(y=None, wp=None, xo=None) == OK and call(taps=1, si=None, so=None) == OK
    assert call(xo=A) == STRIDE and call(so=A) == STRIDE            # long calls are not in place
    assert call(x=None) == NUL and call(xo=None) == NUL and call(wp=None) == OK and call(si=None) == NUL
    assert call(dt=3) == DTYPE and call(g=3) == SHAPE and call(W=0) == SHAPE and call(taps=17) == SHAPE and call(taps=0) == SHAPE
    assert call(W=16388, g=1) == SHAPE and call(W=4098, g=1) == SHAPE and call(W=16384, g=1) == OK
    assert call(x=A + 4) == ALIGN and call(B=0) == SHAPE and call(L=0) == SHAPE


def test_latent_norm_arguments(lib):
    def call(**kw):
        d = dict(p=A, ld=100, wq=A, wk=A, q=A, c=A, cap=64, pd=None, pos=60, B=1, L=4, Q=30, R=20, dt=0)
        d.update(kw)
        return lib.pq_validate_latent_norm(*[d[k] for k in ("p", "ld", "wq", "wk", "q", "c", "cap", "pd", "pos", "B", "L", "Q", "R", "dt")])
    assert call() == OK and call(wk=None, c=None, cap=0) == OK
    assert call(pos=61) == STRIDE and call(ld=49) == STRIDE and call(c=None) == NUL and call(dt=5) == DTYPE and call(Q=0) == SHAPE


def test_head_linear_arguments(lib):
    def call(**kw):
        d = dict(x=A, xr=64, xh=32, w=A, g=None, gr=0, y=A, yr=32, yh=16, M=3, H=2, N=16, K=32, e=0, dt=1)
        d.update(kw)
        return lib.pq_validate_head_linear(*[d[k] for k in ("x", "xr", "xh", "w", "g", "gr", "y", "yr", "yh", "M", "H", "N", "K", "e", "dt")])
    assert call() == OK and call(M=0) == SHAPE and call(e=4) == SHAPE and call(e=2) == NUL and call(e=2, g=A, gr=31) == STRIDE
    assert call(e=2, g=A, gr=32) == OK and call(yh=8) == STRIDE and call(dt=9) == DTYPE and call(x=A + 1) == ALIGN


def test_decode_arguments_and_plan(lib):
    need = lib.pq_latent_decode_workspace_bytes(2, 1, 5, 64, 3)
    assert need == (2 * 3 * 5 * 2 + 2 * 3 * 5 * 64) * 4
    def call(**kw):
        d = dict(q=A, c=A, cap=128, sink=A, start=None, pd=None, pos=100, out=A, B=2, L=1, H=5, R=64, S=3, ws=A, n=need, dt=1)
        d.update(kw)
        return lib.pq_validate_latent_decode(*[d[k] for k in ("q", "c", "cap", "sink", "start", "pd", "pos", "out", "B", "L", "H", "R", "S", "ws", "n", "dt")])
    assert call() == OK and call(n=need - 1) == WS and call(S=0) == WS and call(S=513) == WS and call(ws=None) == NUL
    assert call(dt=2, ws=None, n=0) == OK and call(R=36, ws=None, n=0) == OK              # plain kernel: no workspace
    assert call(pos=128) == STRIDE and call(L=28) == WS and call(R=0) == SHAPE and call(sink=None) == NUL and call(q=A + 2) == ALIGN
    for args in ((1, 1, 32, 1), (8, 1, 32, 1 << 17), (1, 16, 128, 10 ** 6), (4096, 1, 1, 5)):
        assert 1 <= lib.pq_latent_decode_plan(*args, 256) <= 512


def test_prefill_arguments(lib):
    def call(**kw):
        d = dict(q=A, k=A, vt=A, ld=128, sink=A, g=None, gr=0, start=None, out=A, B=1, L=20, Lk=100, H=3, D=64, Dv=40, dt=0)
        d.update(kw)
        return lib.pq_validate_latent_prefill(*[d[k] for k in ("q", "k", "vt", "ld", "sink", "g", "gr", "start", "out", "B", "L", "Lk", "H", "D", "Dv", "dt")])
    assert call() == OK and call(ld=100) == STRIDE and call(ld=64) == STRIDE and call(Lk=19) == SHAPE and call(dt=2) == DTYPE
    assert call(D=20) == SHAPE and call(D=264) == SHAPE and call(Dv=257) == SHAPE and call(g=A, gr=119) == STRIDE and call(g=A, gr=120) == OK
    assert lib.pq_latent_prefill_takes(192, 128, 1) == 1 and lib.pq_latent_prefill_takes(192, 128, 2) == 0


def test_ops_refuse_cpu_tensors():
    from polarquant_amd import latent_ops as ops
    with pytest.raises(RuntimeError, match="no CPU fallback"):
        ops.relu_sq(torch.zeros(8))
