"""Latent attention and the layer steps around it, as HIP launches (include/polarquant_latent.h): residual add + grouped
norms + input convolution, the latents' norms with the cache append, per-head products, attention over the latent cache.
float16, bfloat16 or float32 weights and activations; the residual stream and the convolution's state are float32."""
from __future__ import annotations

from typing import Optional, Tuple

import torch

from . import _ffi
from .attention import _num_cus
from .kernel4group import _stream_ptr

_DTYPES = {torch.float16: _ffi.PQ_F16, torch.bfloat16: _ffi.PQ_BF16, torch.float32: _ffi.PQ_F32}
IN_PLACE_TOKENS = 32        # longer calls are cut into strips that read what others of the launch write
SMALL_M = 16                # rows the weight-streaming product kernels take


def _code(t: torch.Tensor) -> int:
    if not t.is_cuda:
        raise RuntimeError("polarquant_amd: the latent-attention ops need tensors on the GPU (no CPU fallback)")
    return _DTYPES[t.dtype]


def _ptr(t: Optional[torch.Tensor]):
    return None if t is None else t.data_ptr()


class ConvState:
    """Inputs of a causal convolution that later tokens still need: float32 [B, taps - 1, width], oldest first.  A call of
    many tokens writes the other of two buffers (its first workgroup reads what its last one writes)."""

    def __init__(self, B: int, taps: int, width: int, device):
        self.taps = taps
        self._buf = [torch.zeros(B, max(taps - 1, 0), width, dtype=torch.float32, device=device) for _ in range(2)]

    @property
    def rows(self) -> torch.Tensor:
        return self._buf[0]

    def targets(self, tokens: int) -> Tuple[torch.Tensor, torch.Tensor]:
        """(read, written) buffers of a call of `tokens` tokens; the written one is `rows` from then on."""
        if tokens <= IN_PLACE_TOKENS:
            return self._buf[0], self._buf[0]
        self._buf.reverse()
        return self._buf[1], self._buf[0]

    def reset(self):
        self._buf[0].zero_()


def norm_conv(x: torch.Tensor, w_pre: torch.Tensor, groups: int, eps: float, y: Optional[torch.Tensor] = None,
              w_post: Optional[torch.Tensor] = None, conv_w: Optional[torch.Tensor] = None, state: Optional[ConvState] = None,
              start: Optional[torch.Tensor] = None, pos: int = 0, pos_dev: Optional[torch.Tensor] = None):
    """x [B, L, W] float32, y [B, L, W] in the dtype -> (x + gnorm(y) w_post, n + conv(n)) with n = gnorm(first) w_pre,
    gnorm normalizing each of `groups` equal parts.  Without y the stream is returned as it is, without conv_w n itself.
    The new stream overwrites x for short calls.  start: int32 [B], positions before it are padding (n = 0)."""
    B, L, W = x.shape
    assert x.is_contiguous() and x.dtype == torch.float32 and w_pre.numel() == W
    dt = _code(w_pre)
    if y is not None:
        assert y.is_contiguous() and y.shape == x.shape and y.dtype == w_pre.dtype == w_post.dtype and w_post.numel() == W
    x_out = None if y is None else (x if L <= IN_PLACE_TOKENS else torch.empty_like(x))
    s_in = s_out = None
    taps = 1
    if conv_w is not None:
        assert conv_w.is_contiguous() and conv_w.shape[0] == W and conv_w.dtype == w_pre.dtype and conv_w.shape[1] == state.taps
        taps = conv_w.shape[1]
        s_in, s_out = state.targets(L)
        assert s_in.shape == (B, taps - 1, W)
    h = torch.empty(B, L, W, dtype=w_pre.dtype, device=x.device)
    with torch.cuda.device(x.device):
        rc = _ffi.latent_lib().pq_norm_conv(
            _ptr(x), _ptr(y), _ptr(w_post) if y is not None else None, _ptr(x_out), _ptr(w_pre), _ptr(conv_w),
            _ptr(s_in) if taps > 1 else None, _ptr(s_out) if taps > 1 else None, _ptr(h), _ptr(start), _ptr(pos_dev), pos, B, L, W,
            groups, taps, float(eps), dt, _stream_ptr(x.device))
    _ffi.check(rc, "pq_norm_conv")
    return (x if y is None else x_out), h


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


def relu_sq(x: torch.Tensor) -> torch.Tensor:
    """max(x, 0)^2, in place."""
    dt = _code(x)
    assert x.is_contiguous()
    with torch.cuda.device(x.device):
        rc = _ffi.latent_lib().pq_relu_sq(_ptr(x), _ptr(x), x.numel(), dt, _stream_ptr(x.device))
    _ffi.check(rc, "pq_relu_sq")
    return x


def head_linear(x: torch.Tensor, w: torch.Tensor, gate: Optional[torch.Tensor] = None, epilogue: int = _ffi.PQ_EPI_PLAIN) -> torch.Tensor:
    """x [M, heads, K], w [heads, N, K] -> [M, heads, N], each head its own product.  gate: [M, heads * N] (rows may be a
    slice of a wider tensor), the result is multiplied by its sigmoid."""
    M, H, K = x.shape
    N = w.shape[1]
    dt = _code(x)
    assert w.is_contiguous() and w.shape == (H, N, K) and w.dtype == x.dtype and x.stride(2) == 1
    if gate is not None:
        assert gate.shape == (M, H * N) and gate.stride(1) == 1 and gate.dtype == x.dtype
        epilogue = _ffi.PQ_EPI_SIGMOID_GATE
    y = torch.empty(M, H, N, dtype=torch.float32 if epilogue == _ffi.PQ_EPI_F32 else x.dtype, device=x.device)
    rows = SMALL_M if (dt != _ffi.PQ_F32 and N % 16 == 0 and K % 32 == 0) else 65535
    with torch.cuda.device(x.device):
        for m in range(0, M, rows):
            xs, ys, gs = x[m:m + rows], y[m:m + rows], None if gate is None else gate[m:m + rows]
            rc = _ffi.latent_lib().pq_head_linear(_ptr(xs), x.stride(0), x.stride(1), _ptr(w), _ptr(gs), 0 if gate is None else gate.stride(0),
                                                  _ptr(ys), H * N, N, xs.shape[0], H, N, K, epilogue, dt, _stream_ptr(x.device))
            _ffi.check(rc, "pq_head_linear")
    return y


def streams(M: int, w: torch.Tensor) -> bool:
    """Whether x [M, K] w^T runs through the weight-streaming kernel instead of the BLAS library."""
    return M <= SMALL_M and w.dtype != torch.float32 and w.is_contiguous() and w.shape[0] % 16 == 0 and w.shape[1] % 32 == 0


def linear(x: torch.Tensor, w: torch.Tensor, relu_squared: bool = False) -> torch.Tensor:
    """x [..., K] w [N, K]^T, optionally through the square of relu."""
    K = w.shape[1]
    M = x.numel() // K
    if streams(M, w):
        y = head_linear(x.reshape(M, 1, K), w.unsqueeze(0), epilogue=_ffi.PQ_EPI_RELU_SQ if relu_squared else _ffi.PQ_EPI_PLAIN)
        return y.view(x.shape[:-1] + (w.shape[0],))
    y = torch.nn.functional.linear(x, w)
    return relu_sq(y) if relu_squared else y


def linear_f32(x: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
    """x [..., K] w^T as float32 (sums that are never rounded to a 16-bit dtype, for up to 64 rows; more rows go through
    the BLAS library, which rounds)."""
    K = w.shape[1]
    M = x.numel() // K
    if M <= 4 * SMALL_M and streams(min(M, SMALL_M), w):
        return head_linear(x.reshape(M, 1, K), w.unsqueeze(0), epilogue=_ffi.PQ_EPI_F32).view(x.shape[:-1] + (w.shape[0],))
    return torch.nn.functional.linear(x, w).float()


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
