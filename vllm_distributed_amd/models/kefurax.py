"""Kefurax: a decoder-only model whose sublayers read an fp32 residual stream un-normed and are normed on their way
OUT, with one of three sequence mixers per layer.

``x = embed[token] * embedding.scale``; per layer ``x <- x + m * norm1(mixer(x))`` and, where the layer has a
feed-forward, ``x <- x + m * norm2(ff(x))`` with ``m = residual_mult``; RMS norms with plain gains.  ``config.json``
lists the layers one by one (``layers[i] = {type, mixer{...}, mlp{...} | null}``), so order, heads, sizes and constants
differ from layer to layer and from model to model.  A final norm and the head give fp32 logits.

Mixers
  * ``rglru`` - ``layers.linear_attention.GatedUnitRecurrence``: two branches ``[y | x]``; x passes a convolution with
    bias, then the real-gated linear recurrence whose gates are block-diagonal projections of its own input; the state
    times ``gelu_tanh(y)`` goes into the output projection.
  * ``mamba1`` - ``layers.linear_attention.ChannelStateSpace``: one projection gives ``[x | z]``; x passes a convolution
    with bias and SiLU and gives ``[dt | B | C]`` through a second projection, dt widened by a third; the selective
    scan's output times ``silu(z)`` goes into the output projection.
  * ``parallel`` - two mixers side by side on the same input (``layers.parallel_heads.ParallelHeads``):
    left = ``layers.attention.WindowBiasAttention`` without window or distance bias, over heads that are rotated
    (neighbouring pairs, YaRN frequencies) and THEN RMS-normed without gain, one added to the softmax denominator, an
    element-wise sigmoid gate; right = ``layers.linear_attention.DeltaRuleMixer`` in its direct form (one decay per head,
    a SiLU gate behind the per-head norm).

Feed-forward: ``layers.moe.GatedMLP`` with the tanh form of GELU.

Tensor and pipeline parallelism are not implemented for this family (the norms reduce over whole rows and the
recurrent state is not sharded).
"""
from __future__ import annotations

from typing import Dict, Iterable, List, Optional, Tuple

import torch
import torch.nn as nn

from .. import ops
from ..config import VllmConfig
from ..parallel.state import get_pp_group, get_tensor_model_parallel_world_size
from .layers.attention import Attention, ResidualRMSNorm, WindowBiasAttention, get_forward_context, rotary_frequencies
from .layers.linear import ColumnParallelLinear, ReplicatedLinear, RowParallelLinear, VocabParallelEmbedding
from .layers.linear_attention import ChannelStateSpace, DeltaRuleMixer, GatedUnitRecurrence
from .layers.moe import GatedMLP
from .layers.parallel_heads import ParallelHeads
from .layers.short_conv import ShortConv, SlotState, conv_rows, stated_taps
from .utils import IntermediateTensors, materialize

Shapes = Dict[str, Tuple[int, ...]]


def _f32(*shape: int) -> nn.Parameter:
    return nn.Parameter(torch.zeros(shape, dtype=torch.float32), requires_grad=False)


def _size(m: dict, key: str, shapes: Shapes, tensor: str, dim: int) -> int:
    """A size the config states, else the checkpoint tensor's ``dim``-th dimension."""
    if m.get(key) is not None:
        return int(m[key])
    shape = shapes.get(tensor)
    if shape is None or dim >= len(shape):
        raise ValueError(f"neither the config ({key}) nor a checkpoint tensor ({tensor}) gives a size")
    return int(shape[dim])


# ---------------------------------------------------------------------------------------------------- mixers
class GatedUnitMixer(nn.Module):
    def __init__(self, width: int, m: dict, layer_idx: int, dtype: torch.dtype, shapes: Shapes):
        super().__init__()
        p = f"l{layer_idx}.mix."
        self.inner = _size(m, "width", shapes, p + "x", 0)
        self.proj = ColumnParallelLinear(width, [self.inner, self.inner], False, dtype)          # [y | x]
        # (the projections' biases join where their outputs are first read: the recurrence's output gate, the
        # convolution's inputs)
        self.x_bias = _f32(self.inner)
        self.conv = ShortConv([self.inner], stated_taps(shapes, p + "conv", m.get("conv")) or 1, dtype, bias=True)
        self.unit = GatedUnitRecurrence(self.inner, _size(m, "blocks", shapes, p + "ra", 0), layer_idx, dtype)
        self.conv_state = SlotState((max(self.conv.taps - 1, 1), self.inner))
        self.unit_state = SlotState(self.unit.per_slot_shape(), torch.float32)
        self.o = RowParallelLinear(self.inner, width, False, dtype)

    def state_layers(self) -> List[SlotState]:
        return [self.conv_state, self.unit_state]

    def forward(self, h: torch.Tensor) -> torch.Tensor:
        ctx = get_forward_context()
        md = ctx.attn_metadata
        yx = self.proj(h)
        x = yx[:, self.inner:]
        if md is None:                    # memory-profiling pass: no state
            return self.o(x.contiguous())
        u = ops.short_conv_act(x, self.inner, self.conv.weight_t, self.conv_state.state, md.state_slots,
                               md.query_start_loc, md.seq_lens, conv_rows(md, ctx.positions), ctx.positions, False,
                               md.num_prefills > 0, self.conv.bias, False, self.x_bias)
        return self.o(self.unit(u, yx[:, :self.inner], self.unit_state.state))


class ChannelScanMixer(nn.Module):
    def __init__(self, width: int, m: dict, layer_idx: int, dtype: torch.dtype, shapes: Shapes):
        super().__init__()
        p = f"l{layer_idx}.mix."
        self.inner = _size(m, "inner", shapes, p + "D", 0)
        self.rank, self.n_state = _size(m, "dt_rank", shapes, p + "dt", 1), _size(m, "state", shapes, p + "A_log", 1)
        self.proj = ColumnParallelLinear(width, [self.inner, self.inner], False, dtype)          # [x | z]
        self.conv = ShortConv([self.inner], stated_taps(shapes, p + "conv", m.get("conv")) or 1, dtype, bias=True)
        # stored [dt | B | C], kept [B | C | dt]: B and C then start on 16-byte borders whatever the rank
        self.x_proj = ColumnParallelLinear(self.inner, [self.n_state, self.n_state, self.rank], False, dtype)
        self.dt_proj = ReplicatedLinear(self.rank, self.inner, False, dtype)
        self.ssm = ChannelStateSpace(self.inner, self.n_state, layer_idx)
        self.conv_state = SlotState((max(self.conv.taps - 1, 1), self.inner))
        self.ssm_state = SlotState(self.ssm.per_slot_shape(), torch.float32)
        self.o = RowParallelLinear(self.inner, width, False, dtype)

    def state_layers(self) -> List[SlotState]:
        return [self.conv_state, self.ssm_state]

    def load_x_proj(self, w: torch.Tensor) -> None:
        assert w.shape[0] == self.rank + 2 * self.n_state, (tuple(w.shape), self.rank, self.n_state)
        dst, n = self.x_proj.weight.data, 2 * self.n_state
        dst[:n].copy_(w[self.rank:])
        dst[n:].copy_(w[:self.rank])

    def forward(self, h: torch.Tensor) -> torch.Tensor:
        ctx = get_forward_context()
        md = ctx.attn_metadata
        xz = self.proj(h)
        if md is None:                    # memory-profiling pass: no state
            return self.o(xz[:, :self.inner].contiguous())
        u = ops.short_conv_act(xz, self.inner, self.conv.weight_t, self.conv_state.state, md.state_slots,
                               md.query_start_loc, md.seq_lens, conv_rows(md, ctx.positions), ctx.positions, True,
                               md.num_prefills > 0, self.conv.bias)
        bcd = self.x_proj(u)
        dt = ops.linear_f32(bcd[:, 2 * self.n_state:], self.dt_proj.weight)
        return self.o(self.ssm(u, dt, bcd, xz[:, self.inner:], self.ssm_state.state))


class RotatedNormAttention(nn.Module):
    """The left half of a parallel mixer; writes ``scale * gated heads`` into the columns it is given."""

    def __init__(self, width: int, m: dict, eps: float, layer_idx: int, dtype: torch.dtype, scale: float):
        super().__init__()
        self.heads, self.kv_heads = int(m["heads"]), int(m.get("kv_heads") or m["heads"])
        self.dim, self.vdim = int(m["dim"]), int(m.get("vdim") or m["dim"])
        if self.heads % self.kv_heads:
            raise ValueError(f"layer {layer_idx}: {self.heads} query heads do not divide over {self.kv_heads} kv heads")
        self.eps, self.out_scale = eps, float(scale)
        qs, ks, vs = self.heads * self.dim, self.kv_heads * self.dim, self.kv_heads * self.vdim
        self.channels, self.out_cols = qs + ks + vs, self.heads * self.vdim
        self.proj = ColumnParallelLinear(width, [qs, ks, vs, self.out_cols], False, dtype)
        rot = m.get("rot") or {}
        dims = int(rot.get("dims", self.dim)) if rot else 0
        if dims > self.dim or dims % 2:
            raise ValueError(f"layer {layer_idx}: {dims} rotated dimensions in heads of {self.dim}")
        freq, self.rot_scale = (rotary_frequencies(dims, float(rot.get("base", 10000.0)), rot.get("scaling")) if dims
                                else (None, 1.0))
        self.register_buffer("inv_freq", freq, persistent=False)
        self.attn = WindowBiasAttention(self.heads, self.dim, self.vdim, self.kv_heads,
                                        float(m.get("scale") or self.dim ** -0.5), layer_idx, distance_bias=False,
                                        sink=0.0)

    def forward(self, h: torch.Tensor, index: int, out: torch.Tensor) -> None:
        ctx = get_forward_context()
        md = ctx.attn_metadata
        x = self.proj(h)
        if md is None:                    # memory-profiling pass: no cache
            out.zero_()
            return
        attn = self.attn
        q = ops.rotate_norm_cache(x, self.heads, self.kv_heads, self.dim, self.vdim, self.inv_freq, self.rot_scale, True,
                                  self.eps, None, None, ctx.positions, attn.k_cache, attn.v_cache, md.slot_mapping)
        ops.sigmoid_mul(attn.forward_cached(q), x[:, self.channels:], self.out_scale, out=out)


class ParallelMixer(ParallelHeads):
    def __init__(self, width: int, m: dict, eps: float, layer_idx: int, dtype: torch.dtype, shapes: Shapes):
        right = dict(m["right"])
        right["conv"] = stated_taps(shapes, f"l{layer_idx}.mix.right.q.conv", right.get("conv")) or 1
        super().__init__(RotatedNormAttention(width, m["left"], eps, layer_idx, dtype, float(m.get("left_scale", 1.0))),
                         DeltaRuleMixer(width, right, eps, layer_idx, dtype, 1, float(m.get("right_scale", 1.0)),
                                        direct=True, silu_gate=True), width, dtype)

    def state_layers(self) -> List[SlotState]:
        return [self.right.conv_states[0], self.right.rule_states[0]]


def _make_mixer(width: int, spec: dict, eps: float, layer_idx: int, dtype: torch.dtype, shapes: Shapes) -> nn.Module:
    kind, m = spec.get("type"), spec["mixer"]
    if kind == "rglru":
        return GatedUnitMixer(width, m, layer_idx, dtype, shapes)
    if kind == "mamba1":
        return ChannelScanMixer(width, m, layer_idx, dtype, shapes)
    if kind == "parallel":
        return ParallelMixer(width, m, eps, layer_idx, dtype, shapes)
    raise ValueError(f"layer {layer_idx}: unknown mixer type {kind!r}")


class KefuraxLayer(nn.Module):
    def __init__(self, width: int, spec: dict, eps: float, mult: float, layer_idx: int, dtype: torch.dtype,
                 shapes: Shapes):
        super().__init__()
        self.mult = mult
        self.mix = _make_mixer(width, spec, eps, layer_idx, dtype, shapes)
        self.norm1 = ResidualRMSNorm(width, eps, dtype)
        mlp = spec.get("mlp")
        self.mlp = None
        if mlp is not None:
            if mlp.get("kind", "dense") != "dense":
                raise ValueError(f"layer {layer_idx}: unknown feed-forward kind {mlp['kind']!r}")
            self.mlp = GatedMLP(width, _size(mlp, "ff", shapes, f"l{layer_idx}.mlp.up", 0), dtype, activation="gelu_tanh")
            self.norm2 = ResidualRMSNorm(width, eps, dtype)

    def forward(self, x: torch.Tensor, h: torch.Tensor, then: Optional[ResidualRMSNorm]) -> torch.Tensor:
        """``x``: fp32 residual stream (updated in place), ``h``: the same numbers in the model dtype.  Returns the
        updated stream in the model dtype, or ``then`` of it.  Every output norm, residual add and what follows it are
        one launch."""
        y = self.mix(h)
        if self.mlp is None:
            return self.norm1.fold(y, x, self.mult, then)
        f = self.mlp(self.norm1.fold(y, x, self.mult))
        return self.norm2.fold(f, x, self.mult, then)


class KefuraxForCausalLM(nn.Module):
    has_request_state = True          # convolutions and recurrent layers remember a state per request: no prefix reuse
    residual_dtype = torch.float32

    def __init__(self, vllm_config: VllmConfig):
        super().__init__()
        mc = vllm_config.model_config
        cfg, dtype = mc.hf_config, mc.torch_dtype
        self.cfg, self.dtype = cfg, dtype
        if get_tensor_model_parallel_world_size() > 1 or get_pp_group().world_size > 1:
            raise NotImplementedError("Kefurax runs on one device: its norms reduce over whole rows and its recurrent "
                                      "state is not sharded")
        self.is_first = self.is_last = True
        from ..config import resolve_model_path
        from .loader import checkpoint_tensor_shapes
        shapes = {} if mc.load_format == "dummy" else checkpoint_tensor_shapes(resolve_model_path(mc.model))
        width, eps = int(cfg["width"]), float((cfg.get("norm") or {}).get("eps", 1e-5))
        specs = cfg["layers"]
        if not specs:
            raise ValueError("a Kefurax model needs at least one layer")
        self.width, self.eps, self.vocab = width, eps, int(cfg["vocab"])
        self.embed_scale = float((cfg.get("embedding") or {}).get("scale", 1.0))
        self.start_layer, self.end_layer = 0, len(specs)
        self.embed = VocabParallelEmbedding(self.vocab, width, dtype)
        mult = float(cfg.get("residual_mult", 1.0))
        self.layers = nn.ModuleList(KefuraxLayer(width, s, eps, mult, i, dtype, shapes) for i, s in enumerate(specs))
        self.final_norm = ResidualRMSNorm(width, eps, dtype)
        self.head = ColumnParallelLinear(width, [self.vocab], False, dtype)
        self.trace_residual: Optional[List[torch.Tensor]] = None      # tests: the residual stream after every layer

    def rebind_buffers(self) -> None:
        return None

    def attention_layers(self) -> List[Attention]:
        return [l.mix.left.attn for l in self.layers if isinstance(l.mix, ParallelMixer)]

    def state_layers(self) -> List[SlotState]:
        out: List[SlotState] = []
        for l in self.layers:
            out += l.mix.state_layers()
        return out

    def forward(self, input_ids, positions, intermediate: Optional[IntermediateTensors] = None):
        x = ops.embed_scaled(input_ids, self.embed.weight, self.embed_scale)
        h = ops.add_rms_norm_to(x, None, None, None, self.eps, self.dtype, normed=False)
        n = len(self.layers)
        for i, layer in enumerate(self.layers):
            h = layer(x, h, self.final_norm if i + 1 == n else None)
            if self.trace_residual is not None:
                self.trace_residual.append(x.clone())
        return h

    def compute_logits(self, hidden: torch.Tensor) -> torch.Tensor:
        return ops.linear_f32(hidden, self.head.weight)[..., :self.vocab]

    # ------------------------------------------------------------ weights
    _RGLRU = {"y": ("proj.weight", 0), "x": ("proj.weight", 1), "y.b": ("unit.gate_bias", None), "x.b": ("x_bias", None),
              "conv": ("conv.weight", None), "conv.b": ("conv.bias", None), "ra": ("unit.ra", None),
              "ra.b": ("unit.ra_bias", None), "ri": ("unit.ri", None), "ri.b": ("unit.ri_bias", None),
              "lam": ("unit.lam", None), "o": ("o.weight", None)}
    _MAMBA = {"in": ("proj.weight", None), "conv": ("conv.weight", None), "conv.b": ("conv.bias", None),
              "x": ("x_proj.weight", "x_proj"), "dt": ("dt_proj.weight", None), "dt.b": ("ssm.dt_bias", None),
              "A_log": ("ssm.a_log", None), "D": ("ssm.d_skip", None), "o": ("o.weight", None)}
    _LEFT = {"q": ("left.proj.weight", 0), "k": ("left.proj.weight", 1), "v": ("left.proj.weight", 2),
             "g": ("left.proj.weight", 3), "o": ("o.weight", ("half", 0))}
    _RIGHT = {"q": ("right.proj.weight", 0), "k": ("right.proj.weight", 1), "v": ("right.proj.weight", 2),
              "g": ("right.proj.weight", 3), "b": ("right.proj.weight", 4), "a": ("right.proj.weight", 5),
              "q.conv": ("right.conv.weight", 0), "k.conv": ("right.conv.weight", 1), "v.conv": ("right.conv.weight", 2),
              "A_log": ("right.rule.a_log", None), "dt_bias": ("right.rule.dt_bias", None),
              "norm": ("right.norm", None), "o": ("o.weight", ("half", 1))}
    _MLP = {"gate": ("mlp.w13", 0), "up": ("mlp.w13", 1), "down": ("mlp.w2", None)}

    def _target(self, name: str):
        """Checkpoint tensor name -> (parameter name, shard of a fused parameter)."""
        top = {"embed": "embed.weight", "final.norm": "final_norm.weight", "head": "head.weight"}
        if name in top:
            return top[name], None
        if not name.startswith("l"):
            return None
        idx, _, rest = name[1:].partition(".")
        if not idx.isdigit() or int(idx) >= len(self.layers):
            return None
        layer, base = self.layers[int(idx)], f"layers.{idx}."
        if rest in ("norm1", "norm2"):
            return base + rest + ".weight", None
        kind, _, leaf = rest.partition(".")
        if kind == "mlp" and layer.mlp is not None and leaf in self._MLP:
            p, shard = self._MLP[leaf]
            return base + p, shard
        if kind != "mix":
            return None
        if isinstance(layer.mix, ParallelMixer):
            half, _, leaf = leaf.partition(".")
            table = {"left": self._LEFT, "right": self._RIGHT}.get(half, {})
        else:
            table = self._RGLRU if isinstance(layer.mix, GatedUnitMixer) else self._MAMBA
        if leaf not in table:
            return None
        p, shard = table[leaf]
        return base + "mix." + p, shard

    def map_weight_name(self, name: str) -> Optional[str]:
        t = self._target(name)
        return None if t is None else t[0]

    def _owns_layer(self, name: str) -> bool:
        return True

    def load_weights(self, weights: Iterable[Tuple[str, torch.Tensor]]) -> List[str]:
        params: Dict[str, nn.Parameter] = dict(self.named_parameters())
        loaded = []
        for name, w in weights:
            t = self._target(name)
            if t is None or t[0] not in params:
                continue
            p, shard = params[t[0]], t[1]
            loader = getattr(p, "weight_loader", None)
            if shard == "x_proj" or isinstance(shard, tuple):      # rows in another order / a run of columns
                mix = self.layers[int(name[1:].partition(".")[0])].mix
                if shard == "x_proj":
                    mix.load_x_proj(materialize(w))
                else:
                    mix.load_output_half(shard[1], materialize(w))
            elif loader is not None:
                loader(p, w, shard)
            else:
                w = materialize(w)
                assert w.numel() == p.numel(), (name, tuple(w.shape), tuple(p.shape))
                p.data.copy_(w.reshape(p.shape))
            loaded.append(name)
        return loaded


def weight_shapes(c: dict) -> Dict[str, Tuple[int, ...]]:
    """Checkpoint tensor names and shapes of a Kefurax config (for the random-weight loader)."""
    width, vocab = int(c["width"]), int(c["vocab"])
    out: Dict[str, Tuple[int, ...]] = {"embed": (vocab, width)}
    for i, spec in enumerate(c["layers"]):
        m, p, q = spec["mixer"], f"l{i}.", f"l{i}.mix."
        out[p + "norm1"] = (width,)
        kind = spec["type"]
        if kind == "rglru":
            w, nb = int(m["width"]), int(m["blocks"])
            for nm in ("y", "x"):
                out[q + nm], out[q + nm + ".b"] = (w, width), (w,)
            out[q + "conv"], out[q + "conv.b"] = (w, int(m.get("conv") or 1)), (w,)
            for nm in ("ra", "ri"):
                out[q + nm], out[q + nm + ".b"] = (nb, w // nb, w // nb), (nb, w // nb)
            out[q + "lam"], out[q + "o"] = (w,), (width, w)
        elif kind == "mamba1":
            inner, rank, n = int(m["inner"]), int(m["dt_rank"]), int(m["state"])
            out[q + "in"], out[q + "conv"], out[q + "conv.b"] = (2 * inner, width), (inner, int(m.get("conv") or 1)), (inner,)
            out[q + "x"], out[q + "dt"], out[q + "dt.b"] = (rank + 2 * n, inner), (inner, rank), (inner,)
            out[q + "A_log"], out[q + "D"], out[q + "o"] = (inner, n), (inner,), (width, inner)
        elif kind == "parallel":
            l, q = m["left"], p + "mix.left."
            heads, kvh, dim = int(l["heads"]), int(l.get("kv_heads") or l["heads"]), int(l["dim"])
            vdim = int(l.get("vdim") or dim)
            out[q + "q"], out[q + "k"], out[q + "v"] = (heads * dim, width), (kvh * dim, width), (kvh * vdim, width)
            out[q + "g"], out[q + "o"] = (heads * vdim, width), (width, heads * vdim)
            r, q = m["right"], p + "mix.right."
            heads, kvh, dim = int(r["heads"]), int(r.get("kv_heads") or r["heads"]), int(r["dim"])
            vdim = int(r.get("vdim") or dim)
            for nm, rows in (("q", kvh * dim), ("k", kvh * dim), ("v", heads * vdim)):
                out[q + nm], out[q + nm + ".conv"] = (rows, width), (rows, int(r.get("conv") or 1))
            out[q + "b"], out[q + "a"], out[q + "A_log"], out[q + "dt_bias"] = (heads, width), (heads, width), (heads,), (heads,)
            out[q + "norm"], out[q + "g"], out[q + "o"] = (vdim,), (heads * vdim, width), (width, heads * vdim)
        else:
            raise ValueError(f"layer {i}: unknown mixer type {kind!r}")
        if spec.get("mlp"):
            ff = int(spec["mlp"]["ff"])
            out[p + "norm2"] = (width,)
            out[p + "mlp.gate"], out[p + "mlp.up"], out[p + "mlp.down"] = (ff, width), (ff, width), (width, ff)
    out["final.norm"], out["head"] = (width,), (vocab, width)
    return out


def random_weight(name: str, shape: Tuple[int, ...], gen: torch.Generator, device, dtype) -> torch.Tensor:
    """A plausible random value for a checkpoint tensor (projections that keep the variance, norm gains around one,
    small biases, decays spread over (0, 1))."""
    def uni(lo: float, hi: float) -> torch.Tensor:
        return lo + (hi - lo) * torch.rand(shape, generator=gen, device=device, dtype=torch.float32)
    leaf = name.rsplit(".", 1)[-1]
    if leaf in ("norm1", "norm2", "norm", "D"):
        w = uni(0.8, 1.2)
    elif leaf == "dt_bias" or name.endswith(".dt.b"):
        w = uni(-5.0, -1.0)
    elif leaf == "b" and not name.endswith("right.b"):
        w = uni(-0.5, 0.5)
    elif leaf == "A_log":
        w = uni(-1.0, 2.0)
    elif leaf == "lam":
        w = uni(-6.0, -2.0)
    elif leaf == "conv":
        w = uni(-0.6, 0.6)
    elif name == "embed":
        w = uni(-1.0, 1.0)
    else:
        s = (3.0 / shape[-1]) ** 0.5
        w = uni(-s, s)
    return w.to(dtype)
