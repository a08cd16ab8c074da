"""Kefurax in float64, written from the equations: one function per mechanism, loops over time wherever the design
has a recurrence or a convolution, whole score matrices for attention.  No code is shared with the package.
``w``: checkpoint tensor name -> tensor (any float type; read as float64)."""
import math
from typing import Dict, List, Optional

import torch

F64 = torch.float64


def f64(t):
    return t.to(F64)


def unit_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


def silu(z):
    return z * sigmoid(z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def softplus(z):
    return torch.where(z > 30, z, torch.log1p(torch.exp(torch.clamp(z, max=30.0))))


def causal_conv(h, taps_w, bias=None):
    """``h[T, C]``, ``taps_w[C, taps]`` (newest tap last); taps that reach in front of the first token add nothing."""
    t, taps = h.shape[0], taps_w.shape[1]
    y = torch.zeros_like(h)
    for i in range(t):
        for j in range(taps):
            src = i - (taps - 1) + j
            if src >= 0:
                y[i] += taps_w[:, j] * h[src]
    return y if bias is None else y + bias


# ------------------------------------------------------------------------------------------ gated linear unit recurrence
def gated_unit_scan(log_a, drive, state=None):
    """``S_t = a S + sqrt(1 - a^2) drive`` per channel, ``a = exp(log_a)``: all the states ``[T, W]`` and the last."""
    s = torch.zeros(log_a.shape[1], dtype=log_a.dtype) if state is None else state.clone()
    out = torch.zeros_like(drive)
    for i in range(log_a.shape[0]):
        a = torch.exp(log_a[i])
        s = a * s + torch.sqrt(1.0 - a * a) * drive[i]
        out[i] = s
    return out, s


def gated_unit_gates(u, w, p, blocks):
    """Retention and input gate of every channel: each of ``blocks`` equal runs of channels through its own matrices."""
    t, width = u.shape
    n = width // blocks
    r, i = torch.zeros_like(u), torch.zeros_like(u)
    for b in range(blocks):
        part = u[:, b * n:(b + 1) * n]
        r[:, b * n:(b + 1) * n] = sigmoid(part @ f64(w[p + "ra"])[b].T + f64(w[p + "ra.b"])[b])
        i[:, b * n:(b + 1) * n] = sigmoid(part @ f64(w[p + "ri"])[b].T + f64(w[p + "ri.b"])[b])
    return r, i


def rglru_mixer(h, w, p, m, eps):
    y = gelu_tanh(h @ f64(w[p + "y"]).T + f64(w[p + "y.b"]))
    u = causal_conv(h @ f64(w[p + "x"]).T + f64(w[p + "x.b"]), f64(w[p + "conv"]), f64(w[p + "conv.b"]))
    r, i = gated_unit_gates(u, w, p, int(m["blocks"]))
    s, _ = gated_unit_scan(-8.0 * r * softplus(f64(w[p + "lam"])), i * u)
    return (s * y) @ f64(w[p + "o"]).T


# ------------------------------------------------------------------------------------------ per-channel selective scan
def channel_scan(x, step, b, c, rate, skip, state=None):
    """``x, step[T, C]``, ``b, c[T, N]``, ``rate[C, N]`` = exp(A_log), ``skip[C]`` -> outputs ``[T, C]`` and the final
    state ``[C, N]``."""
    s = torch.zeros_like(rate) if state is None else state.clone()
    y = torch.zeros_like(x)
    for i in range(x.shape[0]):
        d = step[i].view(-1, 1)
        s = torch.exp(-d * rate) * s + d * x[i].view(-1, 1) * b[i].view(1, -1)
        y[i] = s @ c[i] + skip * x[i]
    return y, s


def mamba1_mixer(h, w, p, m, eps):
    inner, rank, n = int(m["inner"]), int(m["dt_rank"]), int(m["state"])
    xz = h @ f64(w[p + "in"]).T
    x = silu(causal_conv(xz[:, :inner], f64(w[p + "conv"]), f64(w[p + "conv.b"])))
    dbc = x @ f64(w[p + "x"]).T
    step = softplus(dbc[:, :rank] @ f64(w[p + "dt"]).T + f64(w[p + "dt.b"]))
    y, _ = channel_scan(x, step, dbc[:, rank:rank + n], dbc[:, rank + n:], torch.exp(f64(w[p + "A_log"])), f64(w[p + "D"]))
    return (y * silu(xz[:, inner:])) @ f64(w[p + "o"]).T


# ------------------------------------------------------------------------------------------ attention
def rotation(rot):
    """Angular frequencies of the pairs and the factor on cos and sin."""
    dims, base = int(rot["dims"]), float(rot["base"])
    freqs = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    sc = rot.get("scaling")
    if not sc:
        return freqs, 1.0

    def dim_of(turns):
        return dims * math.log(sc["original"] / (2.0 * math.pi * turns)) / (2.0 * math.log(base))
    lo, hi = max(math.floor(dim_of(sc["fast"])), 0), min(math.ceil(dim_of(sc["slow"])), dims - 1)
    out = []
    for i, f in enumerate(freqs):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(f / sc["factor"] * ramp + f * (1.0 - ramp))
    return out, 0.1 * math.log(sc["factor"]) + 1.0


def rotate(x, rot):
    """``x[T, H, D]``, token ``t`` at position ``t``; neighbours paired."""
    freqs, mul = rotation(rot)
    y = x.clone()
    pos = torch.arange(x.shape[0], dtype=x.dtype).view(-1, 1)
    for i, f in enumerate(freqs):
        cos, sin = torch.cos(pos * f) * mul, torch.sin(pos * f) * mul
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        y[..., 2 * i], y[..., 2 * i + 1] = u * cos - v * sin, v * cos + u * sin
    return y


def open_softmax(scores, i_from=0):
    """``scores[T, N]``, row ``i`` seeing ``j <= i + i_from``: weights with one more in the denominator."""
    t, n = scores.shape
    hidden = torch.arange(n).view(1, -1) > torch.arange(t).view(-1, 1) + i_from
    s = scores.masked_fill(hidden, float("-inf"))
    top = torch.clamp(s.max(-1, keepdim=True).values, min=0.0)
    e = torch.exp(s - top)
    return e / (torch.exp(-top) + e.sum(-1, keepdim=True))


def attention_heads(h, w, p, m, eps):
    t = h.shape[0]
    heads, groups = int(m["heads"]), int(m.get("kv_heads") or m["heads"])
    dim, vdim = int(m["dim"]), int(m.get("vdim") or m["dim"])
    q = unit_rms(rotate((h @ f64(w[p + "q"]).T).view(t, heads, dim), m["rot"]), eps)
    k = unit_rms(rotate((h @ f64(w[p + "k"]).T).view(t, groups, dim), m["rot"]), eps)
    v = (h @ f64(w[p + "v"]).T).view(t, groups, vdim)
    rep = heads // groups
    o = torch.stack([open_softmax(q[:, i] @ k[:, i // rep].T * float(m["scale"])) @ v[:, i // rep] for i in range(heads)],
                    dim=1).reshape(t, heads * vdim)
    return (o * sigmoid(h @ f64(w[p + "g"]).T)) @ f64(w[p + "o"]).T


# ------------------------------------------------------------------------------------------ gated delta rule
def delta_heads(q, k, v, beta, decay, state=None):
    """``q, k[T, H, D]`` (unit vectors, q scaled), ``v[T, H, V]``, ``beta, decay[T, H]`` -> outputs ``[T, H, V]`` and
    the final state ``[H, D, V]``."""
    t, heads, dim = q.shape
    s = torch.zeros(heads, dim, v.shape[2], dtype=q.dtype) if state is None else state.clone()
    out = torch.zeros_like(v)
    for i in range(t):
        s = decay[i].view(-1, 1, 1) * s
        u = beta[i].view(-1, 1) * (v[i] - torch.einsum("hdv,hd->hv", s, k[i]))
        s = s + k[i].unsqueeze(2) * u.unsqueeze(1)
        out[i] = torch.einsum("hdv,hd->hv", s, q[i])
    return out, s


def delta_mixer(h, w, p, m, eps):
    t = h.shape[0]
    heads, groups = int(m["heads"]), int(m.get("kv_heads") or m["heads"])
    dim, vdim = int(m["dim"]), int(m.get("vdim") or m["dim"])
    q = silu(causal_conv(h @ f64(w[p + "q"]).T, f64(w[p + "q.conv"]))).view(t, groups, dim)
    k = silu(causal_conv(h @ f64(w[p + "k"]).T, f64(w[p + "k.conv"]))).view(t, groups, dim)
    v = silu(causal_conv(h @ f64(w[p + "v"]).T, f64(w[p + "v.conv"]))).view(t, heads, vdim)
    q = q / torch.sqrt((q * q).sum(-1, keepdim=True) + 1e-6) * dim ** -0.5
    k = k / torch.sqrt((k * k).sum(-1, keepdim=True) + 1e-6)
    rep = heads // groups
    beta = sigmoid(h @ f64(w[p + "b"]).T)
    decay = torch.exp(-torch.exp(f64(w[p + "A_log"])) * softplus(h @ f64(w[p + "a"]).T + f64(w[p + "dt_bias"])))
    o, _ = delta_heads(q.repeat_interleave(rep, 1), k.repeat_interleave(rep, 1), v, beta, decay)
    o = unit_rms(o, eps) * f64(w[p + "norm"]) * silu(h @ f64(w[p + "g"]).T).view(t, heads, vdim)
    return o.reshape(t, heads * vdim) @ f64(w[p + "o"]).T


def parallel_mixer(h, w, p, m, eps):
    return (float(m["left_scale"]) * attention_heads(h, w, p + "left.", m["left"], eps)
            + float(m["right_scale"]) * delta_mixer(h, w, p + "right.", m["right"], eps))


# ------------------------------------------------------------------------------------------ the model
def feed_forward(h, w, p):
    return (gelu_tanh(h @ f64(w[p + "gate"]).T) * (h @ f64(w[p + "up"]).T)) @ f64(w[p + "down"]).T


MIXERS = {"rglru": rglru_mixer, "mamba1": mamba1_mixer, "parallel": parallel_mixer}


def forward(cfg: dict, w: Dict[str, torch.Tensor], tokens: List[int], residuals: Optional[list] = None):
    """Logits ``[T, vocab]`` of a whole sequence; ``residuals`` collects the stream after every layer."""
    eps, mult = float(cfg["norm"]["eps"]), float(cfg["residual_mult"])
    x = f64(w["embed"])[tokens] * float(cfg["embedding"]["scale"])
    for i, spec in enumerate(cfg["layers"]):
        p = f"l{i}."
        x = x + mult * unit_rms(MIXERS[spec["type"]](x, w, p + "mix.", spec["mixer"], eps), eps) * f64(w[p + "norm1"])
        if spec.get("mlp"):
            x = x + mult * unit_rms(feed_forward(x, w, p + "mlp."), eps) * f64(w[p + "norm2"])
        if residuals is not None:
            residuals.append(x.clone())
    return (unit_rms(x, eps) * f64(w["final.norm"])) @ f64(w["head"]).T
