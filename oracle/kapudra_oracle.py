"""Plain implementation of the Kapudra decoder, one function per mechanism, in float64 on the CPU.
TEST INFRASTRUCTURE ONLY: written from the design's equations, it shares no code with polarquant_amd/ and is
slow on purpose (no cache: every call runs whole sequences from their first token).

Notation: x[t] the residual stream, h what a layer's mixer and feed-forward read.  `weights` maps tensor names to
tensors, `cfg` is the dict of config.json.
"""
from __future__ import annotations

import math
from typing import Dict, List, Optional, Sequence, Tuple

import torch

F64 = torch.float64


def rms_norm(x: torch.Tensor, w: Optional[torch.Tensor], eps: float) -> torch.Tensor:
    """x / sqrt(mean(x^2) + eps), times w if there is one, over the last dimension."""
    n = x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)
    return n if w is None else n * w


def unit(x: torch.Tensor) -> torch.Tensor:
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def silu(x: torch.Tensor) -> torch.Tensor:
    return x / (1.0 + torch.exp(-x))


def gelu_tanh(x: torch.Tensor) -> torch.Tensor:
    return 0.5 * x * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (x + 0.044715 * x ** 3)))


def softplus(x: torch.Tensor) -> torch.Tensor:
    return torch.clamp(x, min=0.0) + torch.log1p(torch.exp(-x.abs()))


def log_sigmoid(x: torch.Tensor) -> torch.Tensor:
    return -softplus(-x)


def cap(x: torch.Tensor, c: float) -> torch.Tensor:
    return c * torch.tanh(x / c)


def causal_conv(x: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
    """x [T, channels], w [channels, taps]: channel by channel over time, the last tap meets the current token."""
    T, taps = x.shape[0], w.shape[1]
    out = torch.zeros_like(x)
    for t in range(T):
        for j in range(taps):
            s = t - (taps - 1) + j
            if s >= 0:
                out[t] += w[:, j] * x[s]
    return out


def distance_slopes(heads: int) -> torch.Tensor:
    return torch.tensor([2.0 ** (-8.0 * (h + 1) / heads) for h in range(heads)], dtype=F64)


def window_attention(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, scale: float, slopes: torch.Tensor, window: Optional[int]) -> torch.Tensor:
    """q [T, H, d], k [T, G, d], v [T, G, dv]: query i sees keys i - window < j <= i with scores q.k scale - slope (i - j).
    -> [T, H * dv]."""
    T, H, _ = q.shape
    per = H // k.shape[1]
    out = torch.zeros(T, H, v.shape[-1], dtype=q.dtype)
    for i in range(T):
        lo = 0 if window is None else max(0, i - window + 1)
        back = (i - torch.arange(lo, i + 1)).to(q.dtype)
        for h in range(H):
            s = k[lo:i + 1, h // per] @ q[i, h] * scale - slopes[h] * back
            out[i, h] = torch.softmax(s, 0) @ v[lo:i + 1, h // per]
    return out.reshape(T, -1)


def window_attention_fast(q, k, v, scale, slopes, window):
    """`window_attention` with matrix products (compared with it by the tests)."""
    T, H, _ = q.shape
    per = H // k.shape[1]
    back = torch.arange(T)[:, None] - torch.arange(T)[None, :]
    seen = (back >= 0) & (back < (T if window is None else window))
    s = torch.einsum("ihd,jhd->hij", q, k.repeat_interleave(per, 1)) * scale - slopes[:, None, None] * back.to(q.dtype)
    p = torch.softmax(s.masked_fill(~seen, -math.inf), -1)
    return torch.einsum("hij,jhd->ihd", p, v.repeat_interleave(per, 1)).reshape(T, -1)


def delta_rule(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, g: torch.Tensor, beta: torch.Tensor) -> torch.Tensor:
    """q, k [T, Hk, d], v [T, H, dv], g [T, H, d] decays of the state's rows, beta [T, H] -> o [T, H, dv]."""
    T, H, dv = v.shape
    per = H // k.shape[1]
    out = torch.zeros_like(v)
    for h in range(H):
        S = torch.zeros(k.shape[-1], dv, dtype=v.dtype)
        for t in range(T):
            kt, qt = k[t, h // per], q[t, h // per]
            S = g[t, h][:, None] * S
            u = beta[t, h] * (v[t, h] - S.T @ kt)
            S = S + kt[:, None] * u[None, :]
            out[t, h] = S.T @ qt
    return out


def matrix_memory(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, log_i: torch.Tensor, log_f: torch.Tensor) -> torch.Tensor:
    """q, k [T, H, d], v [T, H, dv], log gates [T, H] -> o [T, H, dv]; exponentials relative to a running maximum that
    begins at 0."""
    T, H, dv = v.shape
    out = torch.zeros_like(v)
    for h in range(H):
        S, n, m = torch.zeros(k.shape[-1], dv, dtype=v.dtype), torch.zeros(k.shape[-1], dtype=v.dtype), 0.0
        for t in range(T):
            i, f = float(log_i[t, h]), float(log_f[t, h])
            new = max(f + m, i)
            a, b = math.exp(f + m - new), math.exp(i - new)
            S = a * S + b * k[t, h][:, None] * v[t, h][None, :]
            n = a * n + b * k[t, h]
            m = new
            out[t, h] = (S.T @ q[t, h]) / (max(abs(float(n @ q[t, h])), math.exp(-m)) + 1e-6)
    return out


def left_mixer(h, m, w, p, eps, slow):
    T, H, G = h.shape[0], m["heads"], m["kv_heads"]
    q = rms_norm(h @ w[p + "q"].T, w[p + "q.norm"], eps).view(T, H, m["dim"])
    k = rms_norm(h @ w[p + "k"].T, w[p + "k.norm"], eps).view(T, G, m["dim"])
    v = (h @ w[p + "v"].T).view(T, G, m["vdim"])
    window = m["mask"]["size"] if m.get("mask") else None
    o = (window_attention if slow else window_attention_fast)(q, k, v, m["scale"], distance_slopes(H), window)
    return o @ w[p + "o"].T


def right_mixer(h, m, w, p, eps):
    T, H, G = h.shape[0], m["heads"], m["kv_heads"]
    conv = lambda n: silu(causal_conv(h @ w[p + n].T, w[p + n + ".conv"]))
    q = unit(conv("q").view(T, G, m["dim"])) * m["dim"] ** -0.5
    k = unit(conv("k").view(T, G, m["dim"]))
    v = conv("v").view(T, H, m["vdim"])
    beta = torch.sigmoid(h @ w[p + "b"].T)
    a = softplus(h @ w[p + "a1"].T @ w[p + "a2"].T + w[p + "dt_bias"]).view(T, H, m["dim"])
    g = torch.exp(-torch.exp(w[p + "A_log"])[:, None] * a)
    o = rms_norm(delta_rule(q, k, v, g, beta), w[p + "norm"], eps).reshape(T, -1)
    return (o * torch.sigmoid(h @ w[p + "g1"].T @ w[p + "g2"].T)) @ w[p + "o"].T


def mixer_parallel(h, m, w, p, eps, slow=False):
    return m["left_scale"] * left_mixer(h, m["left"], w, p + "left.", eps, slow) + m["right_scale"] * right_mixer(h, m["right"], w, p + "right.", eps)


def mixer_mlstm(h, m, w, p, eps):
    T, H = h.shape[0], m["heads"]
    q = (h @ w[p + "q"].T).view(T, H, -1) * m["dim"] ** -0.5
    k = (h @ w[p + "k"].T).view(T, H, -1)
    v = (h @ w[p + "v"].T).view(T, H, -1)
    log_i = cap(h @ w[p + "i"].T + w[p + "i.b"], m["gate_cap"])
    log_f = log_sigmoid(cap(h @ w[p + "f"].T + w[p + "f.b"], m["gate_cap"]))
    o = rms_norm(matrix_memory(q, k, v, log_i, log_f), None, eps).reshape(T, -1) * w[p + "norm"]
    return (o * torch.sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


def feed_forward(h, w, p):
    return (gelu_tanh(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def schedule(cfg: Dict) -> List[Tuple[int, Optional[int]]]:
    """(layer, number of the pass that begins with it or None) in the order of running."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    out = [(i, None) for i in range(loop["start"])]
    for t in range(loop["times"]):
        out += [(i, t if i == loop["start"] else None) for i in range(loop["start"], loop["stop"])]
    return out + [(i, None) for i in range(loop["stop"], n)]


def forward(tokens: Sequence[int], cfg: Dict, weights: Dict[str, torch.Tensor], slow: bool = False,
            capture: Optional[List[torch.Tensor]] = None) -> torch.Tensor:
    """Logits [T, vocab] of one sequence; `capture` receives the residual stream after every layer run."""
    w = {k: v.to(F64) for k, v in weights.items()}
    eps = cfg["norm"]["eps"]
    e = w["embed"][torch.as_tensor(list(tokens), dtype=torch.long)] * cfg["embedding"]["scale"]
    x = e
    for i, begins in schedule(cfg):
        if begins is not None:
            x = x + (e if begins > 0 else 0.0) + w["loop.step"][begins]
        layer, l = cfg["layers"][i], "l%d." % i
        h = rms_norm(x, w[l + "norm1"], eps)
        if layer["type"] == "parallel":
            y = mixer_parallel(h, layer["mixer"], w, l + "mix.", eps, slow)
        else:
            y = mixer_mlstm(h, layer["mixer"], w, l + "mix.", eps)
        if layer.get("mlp") is not None:
            y = y + feed_forward(h, w, l + "mlp.")
        x = x + y
        if capture is not None:
            capture.append(x.clone())
    z = rms_norm(x, w["final.norm"], eps) @ w["head"].T * cfg["logit_scale"]
    return cap(z, cfg["logit_softcap"])


def tensor_shapes(cfg: Dict, decay_rank: int = 12, gate_rank: int = 20) -> Dict[str, Tuple[int, ...]]:
    """Every tensor name of a model with configuration `cfg`, with its shape; the ranks of the two low-rank products of a
    delta-rule mixer are the caller's choice (a checkpoint's shapes give them)."""
    W, out = cfg["width"], {"embed": (cfg["vocab"], cfg["width"])}
    if cfg.get("loop"):
        out["loop.step"] = (cfg["loop"]["times"], W)
    for i, layer in enumerate(cfg["layers"]):
        m, l = layer["mixer"], "l%d." % i
        out[l + "norm1"] = (W,)
        if layer["type"] == "parallel":
            a, p = m["left"], l + "mix.left."
            qd, kd = a["heads"] * a["dim"], a["kv_heads"] * a["dim"]
            out.update({p + "q": (qd, W), p + "k": (kd, W), p + "v": (a["kv_heads"] * a["vdim"], W), p + "q.norm": (qd,), p + "k.norm": (kd,),
                        p + "o": (W, a["heads"] * a["vdim"])})
            a, p = m["right"], l + "mix.right."
            kd, gd, vd = a["kv_heads"] * a["dim"], a["heads"] * a["dim"], a["heads"] * a["vdim"]
            for n, d in (("q", kd), ("k", kd), ("v", vd)):
                out.update({p + n: (d, W), p + n + ".conv": (d, a["conv"])})
            out.update({p + "b": (a["heads"], W), p + "A_log": (a["heads"],), p + "norm": (a["vdim"],), p + "a1": (decay_rank, W), p + "a2": (gd, decay_rank),
                        p + "dt_bias": (gd,), p + "g1": (gate_rank, W), p + "g2": (vd, gate_rank), p + "o": (W, vd)})
        else:
            p, qd, vd = l + "mix.", m["heads"] * m["dim"], m["heads"] * m["vdim"]
            out.update({p + "q": (qd, W), p + "k": (qd, W), p + "v": (vd, W), p + "g": (vd, W), p + "o": (W, vd), p + "norm": (vd,),
                        p + "i": (m["heads"], W), p + "i.b": (m["heads"],), p + "f": (m["heads"], W), p + "f.b": (m["heads"],)})
        if layer.get("mlp") is not None:
            F = layer["mlp"]["ff"]
            out.update({l + "mlp.gate": (F, W), l + "mlp.up": (F, W), l + "mlp.down": (W, F)})
    out.update({"final.norm": (W,), "head": (cfg["vocab"], W)})
    return out


def random_weights(cfg: Dict, seed: int, dtype=torch.bfloat16, **ranks) -> Dict[str, torch.Tensor]:
    """Weights that keep activations near unit size, slow and fast decays, open and shut gates."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(cfg, **ranks).items():
        r = torch.randn(shape, generator=g, dtype=torch.float32)
        if name.endswith("norm") or name.endswith("norm1"):
            r = 1.0 + 0.2 * r
        elif name.endswith(".conv"):
            r = 0.6 * r
        elif name.endswith("A_log"):
            r = 1.2 * r - 1.5
        elif name.endswith("dt_bias"):
            r = r - 1.0
        elif name.endswith("i.b"):
            r = 1.5 * r
        elif name.endswith("f.b"):
            r = 3.0 + 1.5 * r
        elif name == "loop.step":
            r = 0.3 * r
        elif name == "embed":
            r = r / cfg["embedding"]["scale"]
        else:
            r = r / math.sqrt(shape[-1])
        out[name] = r.to(dtype)
    return out
