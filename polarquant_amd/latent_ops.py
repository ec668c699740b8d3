"""Latent attention as HIP launches (include/polarquant_latent.h): the latents' norms with the cache append, attention over
the latent cache; with the layer steps of `layer_ops`.  float16, bfloat16 or float32 weights and activations."""
from __future__ import annotations

from typing import Optional

import torch

from . import _ffi
from .attention import _num_cus
from .kernel4group import _stream_ptr

from .layer_ops import (_DTYPES, _code, _ptr, ConvState, IN_PLACE_TOKENS, SMALL_M, head_linear, linear, linear_f32,  # noqa: F401
                        norm_conv, relu_sq, streams)


def latent_norm(p: torch.Tensor, w_q: torch.Tensor, w_kv: Optional[torch.Tensor], cache: Optional[torch.Tensor], eps: float,
                pos: int, pos_dev: Optional[torch.Tensor] = None) -> torch.Tensor:
    """p [B, L, >= q_rank + kv_rank] (projection output) -> normed query latent [B, L, q_rank]; the normed key/value latent
    goes to rows pos .. of cache [B, capacity, kv_rank]."""
    B, L, ld = p.shape
    dt = _code(p)
    assert p.is_contiguous() and w_q.dtype == p.dtype and (w_kv is None or (w_kv.dtype == p.dtype and cache.dtype == p.dtype))
    assert cache is None or (cache.is_contiguous() and cache.shape[0] == B and (w_kv is None or cache.shape[2] == w_kv.numel()))
    qr = w_q.numel()
    out = torch.empty(B, L, qr, dtype=p.dtype, device=p.device)
    with torch.cuda.device(p.device):
        rc = _ffi.latent_lib().pq_latent_norm(_ptr(p), ld, _ptr(w_q), _ptr(w_kv), _ptr(out), _ptr(cache) if w_kv is not None else None,
                                              cache.shape[1] if w_kv is not None else 0, _ptr(pos_dev), pos, B, L, qr,
                                              w_kv.numel() if w_kv is not None else 1, float(eps), dt, _stream_ptr(p.device))
    _ffi.check(rc, "pq_latent_norm")
    return out


def decode_splits(B: int, L: int, H: int, max_keys: int, device) -> int:
    return _ffi.latent_lib().pq_latent_decode_plan(B, L, H, max_keys, _num_cus(device))


def latent_decode_attention(q: torch.Tensor, cache: torch.Tensor, sink: torch.Tensor, scale: float, pos: int,
                            pos_dev: Optional[torch.Tensor] = None, start: Optional[torch.Tensor] = None,
                            n_splits: Optional[int] = None) -> torch.Tensor:
    """q [B, L, H, R] in the latent space, cache [B, capacity, R] shared by the heads, rows [0, pos + L) filled; query t
    sees keys start[b] <= j <= pos + t.  -> [B, L, H, R].  With pos_dev, n_splits must be given (the host does not know
    the length)."""
    B, L, H, R = q.shape
    dt = _code(q)
    assert q.is_contiguous() and cache.is_contiguous() and cache.shape[0] == B and cache.shape[2] == R and cache.dtype == q.dtype
    assert sink.dtype == torch.float32 and sink.numel() == H and sink.is_contiguous()
    if n_splits is None:
        assert pos_dev is None
        n_splits = decode_splits(B, L, H, pos + L, q.device)
    lib = _ffi.latent_lib()
    nbytes = lib.pq_latent_decode_workspace_bytes(B, L, H, R, n_splits)
    ws = torch.empty(nbytes // 4, dtype=torch.float32, device=q.device) if dt != _ffi.PQ_F32 else None
    out = torch.empty_like(q)
    with torch.cuda.device(q.device):
        rc = lib.pq_latent_decode(_ptr(q), _ptr(cache), cache.shape[1], _ptr(sink), _ptr(start), _ptr(pos_dev), pos, _ptr(out), B, L, H,
                                  R, float(scale), n_splits, _ptr(ws), nbytes if ws is not None else 0, dt, _stream_ptr(q.device))
    _ffi.check(rc, "pq_latent_decode")
    return out


def prefill_takes(dim: int, vdim: int, dtype: torch.dtype) -> bool:
    return bool(_ffi.latent_lib().pq_latent_prefill_takes(dim, vdim, _DTYPES[dtype]))


def latent_prefill_attention(q: torch.Tensor, k: torch.Tensor, vt: torch.Tensor, sink: torch.Tensor, scale: float,
                             gate: Optional[torch.Tensor] = None, start: Optional[torch.Tensor] = None) -> torch.Tensor:
    """q [B, L, H, D], k [B, Lk, H, D] (the new tokens are the last L of the Lk), vt [B, H, Dv, ld >= Lk] with ld % 64 == 0,
    gate [B * L, H * Dv] (rows may be a slice of a wider tensor) -> softmax(q k^T, sink) v * sigmoid(gate), [B, L, H * Dv]."""
    B, L, H, D = q.shape
    Lk, Dv, ld = k.shape[1], vt.shape[2], vt.shape[3]
    dt = _code(q)
    assert q.is_contiguous() and k.is_contiguous() and vt.is_contiguous() and k.shape == (B, Lk, H, D) and vt.shape[:2] == (B, H)
    assert k.dtype == vt.dtype == q.dtype and sink.dtype == torch.float32 and sink.numel() == H
    if gate is not None:
        assert gate.shape == (B * L, H * Dv) and gate.stride(1) == 1 and gate.dtype == q.dtype
        if gate.data_ptr() % 8:
            gate = gate.contiguous()
    out = torch.empty(B, L, H * Dv, dtype=q.dtype, device=q.device)
    with torch.cuda.device(q.device):
        rc = _ffi.latent_lib().pq_latent_prefill(_ptr(q), _ptr(k), _ptr(vt), ld, _ptr(sink), _ptr(gate), 0 if gate is None else gate.stride(0),
                                                 _ptr(start), _ptr(out), B, L, Lk, H, D, Dv, float(scale), dt, _stream_ptr(q.device))
    _ffi.check(rc, "pq_latent_prefill")
    return out
