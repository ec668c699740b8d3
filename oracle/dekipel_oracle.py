"""Plain implementation of the Dekipel decoder, one function per mechanism, in float64 on the CPU.
TEST INFRASTRUCTURE ONLY: written from the design's equations, it shares no code with polarquant_amd/ and is
slow on purpose (no cache: every call runs whole sequences from their first token).

Notation: x[t] the residual stream, h what a sublayer reads, c the latent key/value state of a token.
`weights` maps tensor names to tensors, `cfg` is the dict of config.json.
"""
from __future__ import annotations

import math
from typing import Dict, List, Optional, Sequence, Tuple

import torch

F64 = torch.float64


def rms_norm(x: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    """w * x / sqrt(mean(x^2) + eps) over the last dimension."""
    return w * x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def grouped_rms_norm(x: torch.Tensor, w: torch.Tensor, eps: float, groups: int) -> torch.Tensor:
    """Each of `groups` equal consecutive parts is divided by its own root mean square; then times w."""
    n = x.shape[-1] // groups
    parts = [x[..., g * n:(g + 1) * n] for g in range(groups)]
    return w * torch.cat([p / torch.sqrt((p * p).mean(-1, keepdim=True) + eps) for p in parts], dim=-1)


def input_conv(h: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
    """h [T, width], w [width, taps] -> h + the causal depthwise convolution whose last tap meets the current token."""
    T, taps = h.shape[0], w.shape[1]
    out = h.clone()
    for t in range(T):
        for j in range(taps):
            s = t - taps + 1 + j
            if s >= 0:
                out[t] = out[t] + w[:, j] * h[s]
    return out


def latent_queries(h: torch.Tensor, w_dq: torch.Tensor, w_norm: torch.Tensor, w_uq: torch.Tensor, eps: float, heads: int) -> torch.Tensor:
    """-> q [T, heads, dim] = W_uq RMSnorm(W_dq h)."""
    return (rms_norm(h @ w_dq.T, w_norm, eps) @ w_uq.T).view(h.shape[0], heads, -1)


def latent_state(h: torch.Tensor, w_dkv: torch.Tensor, w_norm: torch.Tensor, eps: float) -> torch.Tensor:
    """-> c [T, kv_rank]."""
    return rms_norm(h @ w_dkv.T, w_norm, eps)


def sink_softmax(s: torch.Tensor, sink: float) -> torch.Tensor:
    """Weights of the scores s [n]; exp(sink) joins the denominator and nothing else."""
    m = max(float(s.max()), float(sink))
    e = torch.exp(s - m)
    return e / (e.sum() + math.exp(float(sink) - m))


def attend(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, sink: torch.Tensor, scale: float, first: int = 0) -> torch.Tensor:
    """Causal attention, q [Tq, H, d] being the last Tq of the tokens of k [T, H, d], v [T, H, dv]; keys before
    `first` do not exist.  -> [Tq, H * dv]."""
    Tq, H, _ = q.shape
    T = k.shape[0]
    out = torch.zeros(Tq, H, v.shape[-1], dtype=q.dtype)
    for i in range(Tq):
        pos = T - Tq + i
        if pos < first:
            continue
        for h in range(H):
            s = (k[first:pos + 1, h] @ q[i, h]) * scale
            out[i, h] = sink_softmax(s, sink[h]) @ v[first:pos + 1, h]
    return out.reshape(Tq, -1)


def attend_fast(q, k, v, sink, scale):
    """`attend` with matrix products, for long sequences (compared with `attend` by the tests)."""
    Tq, H, _ = q.shape
    T = k.shape[0]
    s = torch.einsum("ihd,jhd->hij", q, k) * scale
    i = torch.arange(Tq)[:, None] + (T - Tq)
    s = s.masked_fill((torch.arange(T)[None, :] > i)[None], -math.inf)
    m = torch.maximum(s.amax(-1, keepdim=True), sink[:, None, None])
    e = torch.exp(s - m)
    p = e / (e.sum(-1, keepdim=True) + torch.exp(sink[:, None, None] - m))
    return torch.einsum("hij,jhd->ihd", p, v).reshape(Tq, -1)


def relu_squared_mlp(h: torch.Tensor, w_up: torch.Tensor, w_down: torch.Tensor) -> torch.Tensor:
    return torch.clamp(h @ w_up.T, min=0.0) ** 2 @ w_down.T


def mixer(i: int, h: torch.Tensor, cfg: Dict, w: Dict[str, torch.Tensor], latents: Dict[int, torch.Tensor], slow: bool = False) -> torch.Tensor:
    m = cfg["layers"][i]["mixer"]
    eps, H, p = cfg["norm"]["eps"], m["heads"], "l%d.mix." % i
    T = h.shape[0]
    q = latent_queries(h, w[p + "dq"], w[p + "dq.norm"], w[p + "uq"], eps, H)
    if m.get("kv_from") is None:
        latents[i] = latent_state(h, w[p + "dkv"], w[p + "dkv.norm"], eps)
        c = latents[i]
    else:
        c = latents[m["kv_from"]]
    k = (c @ w[p + "uk"].T).view(T, H, m["dim"])
    v = (c @ w[p + "uv"].T).view(T, H, m["vdim"])
    o = (attend if slow else attend_fast)(q, k, v, w[p + "sink"], m["scale"])
    o = o * torch.sigmoid(h @ w[p + "g"].T)
    return o @ w[p + "o"].T


def forward(tokens: Sequence[int], cfg: Dict, weights: Dict[str, torch.Tensor], slow: bool = False,
            capture: Optional[List[torch.Tensor]] = None) -> torch.Tensor:
    """Logits [T, vocab] of one sequence; `capture` receives the residual stream after every layer."""
    w = {k: v.to(F64) for k, v in weights.items()}
    eps, groups = cfg["norm"]["eps"], cfg["norm"]["groups"]
    gn = lambda x, name: grouped_rms_norm(x, w[name], eps, groups)
    x = w["embed"][torch.as_tensor(list(tokens), dtype=torch.long)]
    latents: Dict[int, torch.Tensor] = {}
    for i, layer in enumerate(cfg["layers"]):
        l = "l%d." % i
        h = input_conv(gn(x, l + "norm1"), w[l + "canon1"])
        x = x + gn(mixer(i, h, cfg, w, latents, slow), l + "norm1b")
        if layer.get("mlp") is not None:
            h = input_conv(gn(x, l + "norm2"), w[l + "canon2"])
            x = x + gn(relu_squared_mlp(h, w[l + "mlp.up"], w[l + "mlp.down"]), l + "norm2b")
        if capture is not None:
            capture.append(x.clone())
    return gn(x, "final.norm") @ w["head"].T


def tensor_shapes(cfg: Dict) -> Dict[str, Tuple[int, ...]]:
    """Every tensor name of a model with configuration `cfg`, with its shape."""
    W, taps, out = cfg["width"], cfg["canon"]["taps"], {"embed": (cfg["vocab"], cfg["width"])}
    for i, layer in enumerate(cfg["layers"]):
        m, l = layer["mixer"], "l%d." % i
        H, R = m["heads"], m["kv_rank"]
        out.update({l + "norm1": (W,), l + "norm1b": (W,), l + "canon1": (W, taps), l + "mix.dq": (m["q_rank"], W),
                    l + "mix.dq.norm": (m["q_rank"],), l + "mix.uq": (H * m["dim"], m["q_rank"]), l + "mix.uk": (H * m["dim"], R),
                    l + "mix.uv": (H * m["vdim"], R), l + "mix.sink": (H,), l + "mix.g": (H * m["vdim"], W), l + "mix.o": (W, H * m["vdim"])})
        if m.get("kv_from") is None:
            out.update({l + "mix.dkv": (R, W), l + "mix.dkv.norm": (R,)})
        if layer.get("mlp") is not None:
            out.update({l + "norm2": (W,), l + "norm2b": (W,), l + "canon2": (W, taps),
                        l + "mlp.up": (layer["mlp"]["ff"], W), l + "mlp.down": (W, layer["mlp"]["ff"])})
    out.update({"final.norm": (W,), "head": (cfg["vocab"], W)})
    return out


def random_weights(cfg: Dict, seed: int, dtype=torch.bfloat16) -> Dict[str, torch.Tensor]:
    """Weights that keep activations near unit size; norm weights around 1, sinks of both signs."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(cfg).items():
        r = torch.randn(shape, generator=g, dtype=torch.float32)
        if "norm" in name:
            r = 1.0 + 0.2 * r
        elif name.endswith("sink"):
            r = r
        elif "canon" in name:
            r = 0.4 * r
        elif name != "embed":
            r = r / math.sqrt(shape[-1]) * (1.5 if name.endswith((".uq", ".uk")) else 1.0)
        out[name] = r.to(dtype)
    return out
