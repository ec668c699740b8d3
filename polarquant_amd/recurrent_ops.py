"""Windowed attention and recurrent mixers as HIP launches (include/polarquant_recurrent.h).  float16, bfloat16 or float32
weights and activations; scores, recurrent state and everything that enters a recurrence are float32.

Tensors called "rows" are [B * L, columns] with unit column stride: slices of a wider tensor will do."""
from __future__ import annotations

from typing import NamedTuple, Optional

import torch

from . import _ffi
from .attention import _num_cus
from .kernel4group import _stream_ptr
from .layer_ops import _DTYPES, ConvState, _code, _ptr

WINDOW_SMALL = 16          # new tokens per sequence up to which keys go to the ring before they are read
MAX_DIM = 256              # of a recurrent head
MAX_TAPS = 16
CHUNKED_TOKENS = WINDOW_SMALL + 1     # from this many tokens per sequence on, 16-bit recurrences run in chunks on the matrix cores
WORKSPACE_BYTES = 384 << 20         # of a chunked recurrence, at most


class Step(NamedTuple):
    """B sequences' next L tokens, at positions pos .. (*pos_dev .. when given), of sequences that begin at `start`."""
    B: int
    L: int
    pos: int
    pos_dev: Optional[torch.Tensor] = None
    start: Optional[torch.Tensor] = None


def _rows(t: torch.Tensor, M: int, n: int, dtype: torch.dtype) -> None:
    assert t.is_cuda and t.dtype == dtype and t.shape == (M, n) and (n == 1 or t.stride(1) == 1), (t.shape, t.stride(), t.dtype)


def _run(lib_fn, name: str, device, *args) -> None:
    with torch.cuda.device(device):
        rc = lib_fn(*args, _stream_ptr(device))
    _ffi.check(rc, name)


# ----------------------------------------------------------------------------- windowed attention
class WindowRing:
    """The last keys and values of B sequences: [B, G, cap, D] and [B, G, cap, Dv], position j in row j % cap."""

    def __init__(self, B: int, G: int, D: int, Dv: int, window: int, dtype, device):
        self.window, self.cap = window, -(-(window + WINDOW_SMALL - 1) // 64) * 64
        self.k = torch.zeros(B, G, self.cap, D, dtype=dtype, device=device)
        self.v = torch.zeros(B, G, self.cap, Dv, dtype=dtype, device=device)


def qk_norm(q, k, v, w_q, w_k, heads: int, eps: float, ring: WindowRing, step: Step):
    """Norms of q and of k over all their columns -> (q [M, H * D], k [M, G * D] or None); with few tokens k and v go to the
    ring."""
    B, G, cap, D = ring.k.shape
    M, Dv, dt = step.B * step.L, ring.v.shape[3], _code(q)
    assert B == step.B and ring.k.is_contiguous() and ring.v.is_contiguous() and ring.k.dtype == ring.v.dtype == q.dtype
    for t, n in ((q, heads * D), (k, G * D), (v, G * Dv)):
        _rows(t, M, n, q.dtype)
        assert t.stride(0) == q.stride(0)
    assert w_q.numel() == heads * D and w_k.numel() == G * D and w_q.dtype == w_k.dtype == q.dtype and w_q.is_contiguous() and w_k.is_contiguous()
    q_out = torch.empty(M, heads * D, dtype=q.dtype, device=q.device)
    k_out = None if step.L <= WINDOW_SMALL else torch.empty(M, G * D, dtype=q.dtype, device=q.device)
    _run(_ffi.recurrent_lib().pq_qk_norm, "pq_qk_norm", q.device, _ptr(q), _ptr(k), _ptr(v), q.stride(0), _ptr(w_q), _ptr(w_k), _ptr(q_out),
         _ptr(k_out), _ptr(ring.k), _ptr(ring.v), _ptr(step.pos_dev), step.pos, B, step.L, heads, G, D, Dv, cap, float(eps), dt)
    return q_out, k_out


def window_attention(q, ring: WindowRing, slopes: Optional[torch.Tensor], scale: float, step: Step, out: torch.Tensor, out_scale: float = 1.0,
                     k_new=None, v_new=None, n_splits: Optional[int] = None) -> torch.Tensor:
    """q [M, H * D] -> out rows [M, H * Dv] = out_scale * attention over the last `ring.window` positions, scores
    scale q.k - slopes[h] * distance.  k_new, v_new: rows of this call's keys and values, which are then put into the ring;
    without them the ring holds those already."""
    B, G, cap, D = ring.k.shape
    Dv, M, dt = ring.v.shape[3], step.B * step.L, _code(q)
    H = q.shape[1] // D
    assert q.is_contiguous() and q.shape == (M, H * D) and H % G == 0 and B == step.B and q.dtype == ring.k.dtype
    _rows(out, M, H * Dv, q.dtype)
    assert slopes is None or (slopes.dtype == torch.float32 and slopes.numel() == H and slopes.is_contiguous())
    if k_new is not None:
        assert step.pos_dev is None
        _rows(k_new, M, G * D, q.dtype)
        _rows(v_new, M, G * Dv, q.dtype)
    else:
        assert step.L <= WINDOW_SMALL
    lib = _ffi.recurrent_lib()
    if k_new is not None:
        n_splits = 1
    elif n_splits is None:
        n_splits = lib.pq_window_plan(B, step.L, H, G, ring.window, _num_cus(q.device))
    nbytes = lib.pq_window_workspace_bytes(B, step.L, H, Dv, n_splits)
    ws = torch.empty(nbytes // 4, dtype=torch.float32, device=q.device) if nbytes else None
    kr, vr = (0, 0) if k_new is None else (k_new.stride(0), v_new.stride(0))
    _run(lib.pq_window_attn, "pq_window_attn", q.device, _ptr(q), _ptr(ring.k), _ptr(ring.v), _ptr(k_new), kr, _ptr(v_new), vr, _ptr(slopes),
         _ptr(step.start), _ptr(step.pos_dev), step.pos, _ptr(out), out.stride(0), B, step.L, H, G, D, Dv, cap, ring.window, float(scale),
         float(out_scale), n_splits, _ptr(ws), nbytes, dt)
    if k_new is not None:
        _run(lib.pq_ring_append, "pq_ring_append", q.device, _ptr(k_new), kr, _ptr(v_new), vr, _ptr(ring.k), _ptr(ring.v), step.pos, B, step.L,
             G, D, Dv, cap, dt)
    return out


# ----------------------------------------------------------------------------- gated delta rule
def _scan_workspace(delta: bool, dtype: torch.dtype, step: Step, heads: int, dim: int, device) -> Optional[torch.Tensor]:
    if dtype == torch.float32 or step.L < CHUNKED_TOKENS or step.pos_dev is not None:
        return None
    need = lambda tokens: _ffi.recurrent_lib().pq_scan_workspace_bytes(int(delta), step.B, heads, dim, tokens, _DTYPES[dtype])
    return torch.empty(min(need(step.L), max(WORKSPACE_BYTES, need(1))), dtype=torch.uint8, device=device)


class DeltaInputs(NamedTuple):
    q: torch.Tensor             # [M, G * dim] after convolution and silu
    k: torch.Tensor
    v: torch.Tensor             # [M, H * vdim]
    q_inv: torch.Tensor         # [M, G] float32: 1 / length, the query's also times dim^-1/2
    k_inv: torch.Tensor
    log_g: torch.Tensor         # [M, H * dim] float32
    beta: torch.Tensor          # [M, H] float32


def delta_prep(q, k, v, b, a, w_q, w_k, w_v, A_log, dt_bias, conv: ConvState, dim: int, vdim: int, step: Step) -> DeltaInputs:
    """Rows q, k [M, G * dim], v [M, H * vdim], b [M, H] of one projection, a [M, H * dim] decay input -> what the recurrence
    takes.  conv: the convolutions' last inputs, of q, k, v side by side."""
    M, dt, dev = step.B * step.L, _code(q), q.device
    H, G = b.shape[1], q.shape[1] // dim
    for t, n in ((q, G * dim), (k, G * dim), (v, H * vdim), (b, H)):
        _rows(t, M, n, q.dtype)
        assert t.stride(0) == q.stride(0)
    _rows(a, M, H * dim, q.dtype)
    taps = conv.taps
    for w, n in ((w_q, G * dim), (w_k, G * dim), (w_v, H * vdim)):
        assert w.shape == (n, taps) and w.is_contiguous() and w.dtype == q.dtype
    assert A_log.numel() == H and dt_bias.numel() == H * dim and A_log.dtype == dt_bias.dtype == q.dtype and A_log.is_contiguous() and dt_bias.is_contiguous()
    s_in, s_out = conv.targets(step.L)
    assert s_in.shape == (step.B, taps - 1, 2 * G * dim + H * vdim)
    e = lambda n, d: torch.empty(M, n, dtype=d, device=dev)
    r = DeltaInputs(e(G * dim, q.dtype), e(G * dim, q.dtype), e(H * vdim, q.dtype), e(G, torch.float32), e(G, torch.float32),
                    e(H * dim, torch.float32), e(H, torch.float32))
    has = taps > 1
    _run(_ffi.recurrent_lib().pq_delta_prep, "pq_delta_prep", dev, _ptr(q), _ptr(k), _ptr(v), _ptr(b), q.stride(0), _ptr(a), a.stride(0), _ptr(w_q),
         _ptr(w_k), _ptr(w_v), _ptr(A_log), _ptr(dt_bias), _ptr(s_in) if has else None, _ptr(s_out) if has else None, _ptr(r.q), _ptr(r.k),
         _ptr(r.v), _ptr(r.q_inv), _ptr(r.k_inv), _ptr(r.log_g), _ptr(r.beta), _ptr(step.start), _ptr(step.pos_dev), step.pos, step.B, step.L, G, H,
         dim, vdim, taps, dt)
    return r


def delta_scan(x: DeltaInputs, state: torch.Tensor, step: Step) -> torch.Tensor:
    """state [B, H, vdim, dim] float32, advanced in place -> o [M, H * vdim] float32."""
    B, H, vdim, dim = state.shape
    M, dt, G = step.B * step.L, _code(x.q), x.q_inv.shape[1]
    assert state.is_contiguous() and state.dtype == torch.float32 and B == step.B and x.q.shape == (M, G * dim) and x.v.shape == (M, H * vdim)
    assert all(t.is_contiguous() for t in x) and x.log_g.shape == (M, H * dim) and x.beta.shape == (M, H)
    o = torch.empty(M, H * vdim, dtype=torch.float32, device=state.device)
    ws = _scan_workspace(True, x.q.dtype, step, H, dim, state.device)
    _run(_ffi.recurrent_lib().pq_delta_scan, "pq_delta_scan", state.device, _ptr(x.q), _ptr(x.k), _ptr(x.v), _ptr(x.q_inv), _ptr(x.k_inv),
         _ptr(x.log_g), _ptr(x.beta), _ptr(state), _ptr(o), _ptr(step.start), _ptr(step.pos_dev), step.pos, B, step.L, G, H, dim, vdim,
         _ptr(ws), 0 if ws is None else ws.numel(), dt)
    return o


# ----------------------------------------------------------------------------- matrix memory
def memory_gates(i, f, b_i, b_f, cap: float):
    """Rows i, f [M, H] of one projection -> (log input gate, log forget gate), float32 [M, H]."""
    M, H = i.shape
    dt = _code(i)
    _rows(i, M, H, i.dtype)
    _rows(f, M, H, i.dtype)
    assert i.stride(0) == f.stride(0) and b_i.numel() == b_f.numel() == H and b_i.dtype == b_f.dtype == i.dtype
    li, lf = [torch.empty(M, H, dtype=torch.float32, device=i.device) for _ in range(2)]
    _run(_ffi.recurrent_lib().pq_memory_gates, "pq_memory_gates", i.device, _ptr(i), _ptr(f), i.stride(0), _ptr(b_i), _ptr(b_f), _ptr(li), _ptr(lf),
         M, H, float(cap), dt)
    return li, lf


def memory_state(B: int, heads: int, dim: int, vdim: int, device):
    """A matrix memory's state at a sequence's start: matrices with the normalizer as their last row, running maxima (a copy
    for every 16 rows, so that no workgroup of a launch reads what another writes)."""
    return (torch.zeros(B, heads, vdim + 1, dim, dtype=torch.float32, device=device),
            torch.zeros(B, heads, (vdim + 16) // 16, dtype=torch.float32, device=device))


def memory_scan(q, k, v, log_i, log_f, state: torch.Tensor, m: torch.Tensor, q_scale: float, step: Step):
    """Rows q, k [M, H * dim], v [M, H * vdim] of one projection; state [B, H, vdim + 1, dim] and m as memory_state has them, advanced in
    place -> (o [M, H * vdim], den [M, H]) float32."""
    B, H, cols, dim = state.shape
    vdim, M, dt = cols - 1, step.B * step.L, _code(q)
    for t, n in ((q, H * dim), (k, H * dim), (v, H * vdim)):
        _rows(t, M, n, q.dtype)
        assert t.stride(0) == q.stride(0)
    assert state.is_contiguous() and m.is_contiguous() and state.dtype == m.dtype == torch.float32 and m.shape == (B, H, (vdim + 16) // 16) and B == step.B
    assert log_i.shape == log_f.shape == (M, H) and log_i.is_contiguous() and log_f.is_contiguous()
    o = torch.empty(M, H * vdim, dtype=torch.float32, device=q.device)
    den = torch.empty(M, H, dtype=torch.float32, device=q.device)
    ws = _scan_workspace(False, q.dtype, step, H, dim, q.device)
    _run(_ffi.recurrent_lib().pq_memory_scan, "pq_memory_scan", q.device, _ptr(q), _ptr(k), _ptr(v), q.stride(0), _ptr(log_i), _ptr(log_f),
         _ptr(state), _ptr(m), _ptr(o), _ptr(den), float(q_scale), _ptr(step.start), _ptr(step.pos_dev), step.pos, B, step.L, H, dim, vdim,
         _ptr(ws), 0 if ws is None else ws.numel(), dt)
    return o, den


def head_norm_gate(o: torch.Tensor, w: torch.Tensor, gate: torch.Tensor, heads: int, eps: float, out: torch.Tensor, out_scale: float = 1.0,
                   den: Optional[torch.Tensor] = None) -> torch.Tensor:
    """o [M, H * vdim] float32 -> out rows = out_scale * rmsnorm per head of o / den, times w ([vdim] or [H * vdim]), times
    sigmoid(gate rows)."""
    M, n = o.shape
    vdim, dt = n // heads, _code(gate)
    _rows(gate, M, n, gate.dtype)
    _rows(out, M, n, gate.dtype)
    assert o.is_contiguous() and o.dtype == torch.float32 and w.numel() in (vdim, n) and w.is_contiguous() and w.dtype == gate.dtype
    assert den is None or (den.is_contiguous() and den.dtype == torch.float32 and den.shape == (M, heads))
    _run(_ffi.recurrent_lib().pq_head_norm_gate, "pq_head_norm_gate", o.device, _ptr(o), _ptr(den), _ptr(w), 0 if w.numel() == vdim else vdim,
         _ptr(gate), gate.stride(0), _ptr(out), out.stride(0), M, heads, vdim, float(eps), float(out_scale), dt)
    return out
