"""Bapovik in float64, written from the equations: one function per mechanism, a loop over time for the recurrence, whole
score matrices for attention, experts token by token.  No code is shared with the package.
``w``: checkpoint tensor name -> tensor (any float type; read as float64)."""
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


# ------------------------------------------------------------------------------------------ attention
def window_mask(t, size):
    """``[T, T]``: row ``i`` sees itself and the ``size - 1`` tokens in front of it."""
    i, j = torch.arange(t).view(-1, 1), torch.arange(t).view(1, -1)
    return (i - j >= 0) & (i - j < size)


def chunk_mask(t, size):
    """``[T, T]``: row ``i`` sees ``j <= i`` of its own block of ``size`` positions."""
    i, j = torch.arange(t).view(-1, 1), torch.arange(t).view(1, -1)
    return (j <= i) & (i // size == j // size)


def capped(scores, cap):
    return cap * torch.tanh(scores / cap)


def weights_of(scores, seen, open_denominator):
    """Softmax over the seen keys; ``open_denominator``: with one more added to the sum of the exponentials."""
    s = scores.masked_fill(~seen, float("-inf"))
    top = s.max(-1, keepdim=True).values
    if open_denominator:
        top = torch.clamp(top, min=0.0)
    e = torch.exp(s - top)
    total = e.sum(-1, keepdim=True)
    if open_denominator:
        total = total + torch.exp(-top)
    return e / total


def project(h, w, name):
    return h @ f64(w[name]).T + f64(w[name + ".b"])


def keys_values(h, w, p, m):
    t, groups = h.shape[0], int(m["kv_heads"])
    return project(h, w, p + "k").view(t, groups, int(m["dim"])), project(h, w, p + "v").view(t, groups, int(m["vdim"]))


def attend(h, q, k, v, w, p, m, seen, cap=None, open_denominator=False):
    """``q[T, H, D]``, ``k[T, G, D]``, ``v[T, G, V]`` -> the mixer's output: every head's result times its own gate, then
    the output projection."""
    t, heads, rep = q.shape[0], q.shape[1], q.shape[1] // k.shape[1]
    gate = sigmoid(h @ f64(w[p + "g"]).T)
    out = []
    for i in range(heads):
        s = q[:, i] @ k[:, i // rep].T * float(m["scale"])
        if cap is not None:
            s = capped(s, cap)
        out.append(weights_of(s, seen, open_denominator) @ v[:, i // rep] * gate[:, i:i + 1])
    return torch.cat(out, dim=1) @ f64(w[p + "o"]).T


def window_mixer(h, w, p, m, eps, kept):
    """``kept``: layer -> (keys, values) of the layers so far; a layer with ``kv_from`` adds none."""
    t, heads = h.shape[0], int(m["heads"])
    q = project(h, w, p + "q").view(t, heads, int(m["dim"]))
    layer = int(p[1:].split(".")[0])
    if m.get("kv_from") is None:
        kept[layer] = keys_values(h, w, p, m)
    k, v = kept[layer if m.get("kv_from") is None else int(m["kv_from"])]
    return attend(h, q, k, v, w, p, m, window_mask(t, int(m["mask"]["size"])))


def chunked_half(h, w, p, m, eps, kept=None):
    t = h.shape[0]
    q = project(h, w, p + "q").view(t, int(m["heads"]), int(m["dim"]))
    k, v = keys_values(h, w, p, m)
    q, k = unit_rms(q, eps) * f64(w[p + "q.norm"]), unit_rms(k, eps) * f64(w[p + "k.norm"])
    if kept is not None:
        kept[int(p[1:].split(".")[0])] = (k, v)
    return attend(h, q, k, v, w, p, m, chunk_mask(t, int(m["mask"]["size"])), float(m["softcap"]), True)


# ------------------------------------------------------------------------------------------ gated linear attention
def channel_decays(h, w, p, m):
    """One decay per head and key channel ``[T, H, D]``, from a projection through a narrow middle."""
    z = h @ f64(w[p + "a1"]).T @ f64(w[p + "a2"]).T + f64(w[p + "a2.b"])
    return (sigmoid(z) ** (1.0 / float(m["tau"]))).view(h.shape[0], int(m["heads"]), int(m["dim"]))


def decayed_heads(q, k, v, alpha, state=None):
    """``q, k, alpha[T, H, D]``, ``v[T, H, V]`` -> outputs ``[T, H, V]`` and the final state ``[H, D, V]``."""
    t, heads, dim = q.shape
    s = torch.zeros(heads, dim, v.shape[2], dtype=q.dtype) if state is None else state.clone()
    out = torch.zeros_like(v)
    for i in range(t):
        s = alpha[i].unsqueeze(2) * s + k[i].unsqueeze(2) * v[i].unsqueeze(1)
        out[i] = (s * q[i].unsqueeze(2)).sum(1)
    return out, s


def recurrent_half(h, w, p, m, eps):
    t, heads, dim, vdim = h.shape[0], int(m["heads"]), int(m["dim"]), int(m["vdim"])
    q = (h @ f64(w[p + "q"]).T).view(t, heads, dim) * dim ** -0.5
    k = (h @ f64(w[p + "k"]).T).view(t, heads, dim)
    v = (h @ f64(w[p + "v"]).T).view(t, heads, vdim)
    o, _ = decayed_heads(q, k, v, channel_decays(h, w, p, m))
    o = (unit_rms(o, eps) * f64(w[p + "norm"])).reshape(t, heads * vdim)
    return (o * silu(h @ f64(w[p + "g"]).T)) @ f64(w[p + "o"]).T


def parallel_mixer(h, w, p, m, eps, kept=None):
    left = chunked_half(h, w, p + "left.", m["left"], eps, kept)
    right = recurrent_half(h, w, p + "right.", m["right"], eps)
    return 0.5 * (unit_rms(left, eps) * f64(w[p + "left.out"]) + unit_rms(right, eps) * f64(w[p + "right.out"]))


# ------------------------------------------------------------------------------------------ experts
def expert(x, w, p):
    up = torch.clamp(f64(w[p + "up"]) @ x, min=0.0)
    return f64(w[p + "down"]) @ (up * up)


def experts(h, w, p, m):
    """Token by token: the ``top`` largest scores, each chosen expert applied to the token times its score."""
    top = int(m["router"]["top"])
    score = sigmoid(h @ f64(w[p + "router"]).T)
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e in torch.argsort(score[t], descending=True)[:top].tolist():
            out[t] += expert(score[t, e] * h[t], w, f"{p}e{e}.")
    return out


# ------------------------------------------------------------------------------------------ the model
def forward(cfg: dict, w: Dict[str, torch.Tensor], tokens: List[int], residuals: Optional[list] = None):
    """Logits ``[T, vocab]`` of a whole sequence; ``residuals`` collects the stream after every layer."""
    eps = float(cfg["norm"]["eps"])
    x = f64(w["embed"])[tokens]
    kept: dict = {}
    for i, spec in enumerate(cfg["layers"]):
        p, m = f"l{i}.", spec["mixer"]
        h = unit_rms(x, eps) * f64(w[p + "norm1"])
        if spec["type"] == "parallel":
            y = parallel_mixer(h, w, p + "mix.", m, eps, kept)
        else:
            y = window_mixer(h, w, p + "mix.", m, eps, kept)
        if spec.get("mlp"):
            y = y + experts(h, w, p + "mlp.", spec["mlp"])
        x = x + y
        if residuals is not None:
            residuals.append(x.clone())
    return (unit_rms(x, eps) * f64(w["final.norm"])) @ f64(w["head"]).T
