"""The steps between a layer's mixers and matrix products, as HIP launches (include/polarquant_steps.h): residual add +
grouped norms + input convolution, activations, per-head and small-batch products.  float16, bfloat16 or float32 weights and
activations; the residual stream and a convolution's state are float32."""
from __future__ import annotations

from typing import Optional, Tuple

import torch

from . import _ffi
from .kernel4group import _stream_ptr

_DTYPES = {torch.float16: _ffi.PQ_F16, torch.bfloat16: _ffi.PQ_BF16, torch.float32: _ffi.PQ_F32}
IN_PLACE_TOKENS = 32        # longer calls are cut into strips that read what others of the launch write
SMALL_M = 16                # rows the weight-streaming product kernels take


def _code(t: torch.Tensor) -> int:
    if not t.is_cuda:
        raise RuntimeError("polarquant_amd: these ops need tensors on the GPU (no CPU fallback)")
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
    gnorm normalizing each of `groups` equal parts; without w_post x + y.  Without y the stream is returned as it is, without conv_w n itself.
    The new stream overwrites x for short calls.  start: int32 [B], positions before it are padding (n = 0)."""
    B, L, W = x.shape
    assert x.is_contiguous() and x.dtype == torch.float32 and w_pre.numel() == W
    dt = _code(w_pre)
    if y is not None:
        assert y.is_contiguous() and y.shape == x.shape and y.dtype == w_pre.dtype
        assert w_post is None or (w_post.dtype == y.dtype and w_post.numel() == W)
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
        rc = _ffi.steps_lib().pq_norm_conv(
            _ptr(x), _ptr(y), _ptr(w_post) if y is not None else None, _ptr(x_out), _ptr(w_pre), _ptr(conv_w),
            _ptr(s_in) if taps > 1 else None, _ptr(s_out) if taps > 1 else None, _ptr(h), _ptr(start), _ptr(pos_dev), pos, B, L, W,
            groups, taps, float(eps), dt, _stream_ptr(x.device))
    _ffi.check(rc, "pq_norm_conv")
    return (x if y is None else x_out), h


def relu_sq(x: torch.Tensor) -> torch.Tensor:
    """max(x, 0)^2, in place."""
    dt = _code(x)
    assert x.is_contiguous()
    with torch.cuda.device(x.device):
        rc = _ffi.steps_lib().pq_relu_sq(_ptr(x), _ptr(x), x.numel(), dt, _stream_ptr(x.device))
    _ffi.check(rc, "pq_relu_sq")
    return x


def gelu_mul(gate: torch.Tensor, up: torch.Tensor, out: Optional[torch.Tensor] = None) -> torch.Tensor:
    """gelu(gate) * up, the tanh form; [M, cols] each, rows may be slices of wider tensors (gate's and up's of one)."""
    dt = _code(gate)
    M, N = gate.shape
    out = torch.empty(M, N, dtype=gate.dtype, device=gate.device) if out is None else out
    assert up.shape == out.shape == (M, N) and gate.stride() == up.stride() and gate.stride(1) == out.stride(1) == 1
    assert up.dtype == out.dtype == gate.dtype
    with torch.cuda.device(gate.device):
        rc = _ffi.steps_lib().pq_gelu_mul(_ptr(gate), _ptr(up), gate.stride(0), _ptr(out), out.stride(0), M, N, dt, _stream_ptr(gate.device))
    _ffi.check(rc, "pq_gelu_mul")
    return out


def stream_add(x: torch.Tensor, y: Optional[torch.Tensor] = None, e: Optional[torch.Tensor] = None, v: Optional[torch.Tensor] = None,
               dtype: torch.dtype = torch.float32) -> torch.Tensor:
    """x + y + e + v as a new stream; x and e float32 [..., W], y like x and v [W] in the model's dtype."""
    W = x.shape[-1]
    for t in (y, v):
        if t is not None:
            dtype = t.dtype
    assert x.is_contiguous() and x.dtype == torch.float32 and (y is None or (y.is_contiguous() and y.shape == x.shape and y.dtype == dtype))
    assert e is None or (e.is_contiguous() and e.shape == x.shape and e.dtype == torch.float32)
    assert v is None or (v.is_contiguous() and v.numel() == W and v.dtype == dtype)
    _code(x)
    out = torch.empty_like(x)
    with torch.cuda.device(x.device):
        rc = _ffi.steps_lib().pq_stream_add(_ptr(x), _ptr(y), _ptr(e), _ptr(v), _ptr(out), x.numel() // W, W, _DTYPES[dtype], _stream_ptr(x.device))
    _ffi.check(rc, "pq_stream_add")
    return out


def embed_rows(table: torch.Tensor, ids: torch.Tensor, scale: float = 1.0) -> torch.Tensor:
    """table[ids] * scale as float32."""
    dt = _code(table)
    ids = ids.contiguous()
    assert table.is_contiguous() and ids.dtype == torch.int64 and ids.is_cuda
    out = torch.empty(tuple(ids.shape) + (table.shape[1],), dtype=torch.float32, device=table.device)
    with torch.cuda.device(table.device):
        rc = _ffi.steps_lib().pq_embed_rows(_ptr(table), _ptr(ids), float(scale), _ptr(out), ids.numel(), table.shape[1], table.shape[0], dt,
                                            _stream_ptr(table.device))
    _ffi.check(rc, "pq_embed_rows")
    return out


def softcap(x: torch.Tensor, scale: float, cap: Optional[float]) -> torch.Tensor:
    """cap * tanh(x * scale / cap) in place, float32; without a cap x * scale."""
    _code(x)
    assert x.is_contiguous() and x.dtype == torch.float32
    with torch.cuda.device(x.device):
        rc = _ffi.steps_lib().pq_softcap(_ptr(x), x.numel(), float(scale), float(cap or 0.0), _stream_ptr(x.device))
    _ffi.check(rc, "pq_softcap")
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
            rc = _ffi.steps_lib().pq_head_linear(_ptr(xs), x.stride(0), x.stride(1), _ptr(w), _ptr(gs), 0 if gate is None else gate.stride(0),
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
