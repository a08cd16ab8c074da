"""Bapovik: a decoder-only model whose layers add a sequence mixer and a block of experts, both reading ONE normed input, to
an fp32 residual stream.

``x = embed[token]``; per layer ``h = norm1(x)``, ``x <- x + mixer(h) + experts(h)`` (RMS norms with plain gains; a layer may
have no experts).  ``config.json`` lists the layers one by one (``layers[i] = {type, mixer{...}, mlp{...} | null}``), so
order, heads, sizes, masks and constants differ from layer to layer and from model to model.  A final norm and the head
give fp32 logits.  Positions enter nowhere but through the masks and the recurrence.

Mixers
  * ``attention`` - ``GatedHeads``: q, k and v with biases, a sliding window, an ordinary softmax, a sigmoid gate per head.  A
    layer with ``kv_from: j`` has no keys and values: it reads what layer ``j`` cached (a parallel layer: its left half),
    with its own queries and mask.
  * ``parallel`` - ``layers.parallel_heads.ParallelNormed``: two mixers side by side on the same input, each one's output
    RMS-normed, half their sum.  left = ``GatedHeads`` with a head norm on q and k, scores squashed to
    ``cap tanh(s / cap)``, a mask of blocks of positions counted from the sequence's start, one added to the softmax
    denominator; right = ``layers.linear_attention.GatedLinearHeads`` (a decay per key channel, per-head norm, SiLU gate).

Feed-forward: ``layers.moe.PlainTopKMoE`` - experts ``down(relu(up(w h))^2)`` whose INPUT carries the routing weight, the
sigmoid of the chosen router outputs as it comes.

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
from .layers.attention import Attention, ResidualRMSNorm, WindowBiasAttention, get_forward_context
from .layers.linear import ColumnParallelLinear, GroupedColumnLinear, RowParallelLinear, VocabParallelEmbedding
from .layers.linear_attention import GatedLinearHeads
from .layers.moe import PlainTopKMoE
from .layers.parallel_heads import ParallelNormed
from .layers.short_conv import SlotState
from .utils import IntermediateTensors, materialize

Shapes = Dict[str, Tuple[int, ...]]


def _f32(*shape: int) -> nn.Parameter:
    return nn.Parameter(torch.zeros(shape, dtype=torch.float32), requires_grad=False)


def _mask_size(m: dict) -> int:
    return int((m.get("mask") or {}).get("size") or 0)


# ---------------------------------------------------------------------------------------------------- mixers
class GatedHeads(nn.Module):
    """Softmax attention between its input projection and its output projection, for either mixer: ``[q | k | v | gate]``
    (a reader of another layer's keys: ``[q | gate]``) as ``forward`` finds them side by side -> the gated heads.  The
    biases of q, k and v join in the launch that (norms and) caches them."""

    def __init__(self, m: dict, eps: float, layer_idx: int, head_norm: bool = False, chunked: bool = False,
                 sink=False, source: Optional["GatedHeads"] = None):
        super().__init__()
        self.heads, self.kv_heads = int(m["heads"]), int(m.get("kv_heads") or m["heads"])
        self.dim, self.vdim = int(m["dim"]), int(m.get("vdim") or m["dim"])
        if self.heads % self.kv_heads:
            raise ValueError(f"layer {layer_idx}: {self.heads} query heads do not divide over {self.kv_heads} kv heads")
        self.eps = eps
        own = source is None
        qkv = [self.heads * self.dim] + ([self.kv_heads * self.dim, self.kv_heads * self.vdim] if own else [])
        self.sizes, self.out_cols = qkv + [self.heads], self.heads * self.vdim
        self.bias_sizes = qkv
        self.bias = _f32(sum(qkv))
        self.bias.weight_loader = self._load_bias              # type: ignore[attr-defined]
        self.q_norm, self.k_norm = (_f32(self.dim), _f32(self.dim)) if head_norm else (None, None)
        size = _mask_size(m)
        self.attn = WindowBiasAttention(self.heads, self.dim, self.vdim, self.kv_heads,
                                        float(m.get("scale") or self.dim ** -0.5), layer_idx,
                                        window=0 if chunked else size, softcap=m.get("softcap"), distance_bias=False,
                                        sink=sink, chunk=size if chunked else 0,
                                        source=None if own else source.attn)

    def _load_bias(self, param: nn.Parameter, w: torch.Tensor, shard_id: int) -> None:
        lo = sum(self.bias_sizes[:shard_id])
        dst = param.data[lo:lo + self.bias_sizes[shard_id]]
        assert tuple(w.shape) == tuple(dst.shape), (tuple(w.shape), tuple(dst.shape))
        dst.copy_(materialize(w))

    def forward(self, x: torch.Tensor) -> torch.Tensor:
        ctx = get_forward_context()
        md = ctx.attn_metadata
        if md is None:                    # memory-profiling pass: no cache
            return x.new_zeros((x.shape[0], self.out_cols))
        attn = self.attn
        own = attn.source is None
        q = ops.rotate_norm_cache(x, self.heads, self.kv_heads if own else 0, self.dim, self.vdim, None, 1.0, False, self.eps,
                                  self.q_norm, self.k_norm, ctx.positions, attn.k_cache if own else None,
                                  attn.v_cache if own else None, md.slot_mapping if own else None,
                                  self.q_norm is not None, self.bias)
        lo = sum(self.bias_sizes)
        return attn.forward_cached(q, x[:, lo:lo + self.heads])


class AttentionMixer(nn.Module):
    def __init__(self, width: int, m: dict, eps: float, layer_idx: int, dtype: torch.dtype,
                 source: Optional[GatedHeads]):
        super().__init__()
        self.inner = GatedHeads(m, eps, layer_idx, source=source)
        self.proj = GroupedColumnLinear(width, [self.inner.sizes], dtype)
        self.o = RowParallelLinear(self.inner.out_cols, width, False, dtype)

    def forward(self, h: torch.Tensor) -> torch.Tensor:
        return self.o(self.inner(self.proj(h)))


def _parallel(width: int, m: dict, eps: float, layer_idx: int, dtype: torch.dtype, shapes: Shapes) -> ParallelNormed:
    r = m["right"]
    rank = r.get("decay_rank")
    if rank is None:                      # the width of the decay's narrow middle is a size only the tensors state
        shape = shapes.get(f"l{layer_idx}.mix.right.a1")
        if shape is None:
            raise ValueError(f"layer {layer_idx}: neither the config (decay_rank) nor a checkpoint tensor (mix.right.a1) "
                             "gives the width of the decay's low-rank projection")
        rank = shape[0]
    left = GatedHeads(m["left"], eps, layer_idx, head_norm=True, chunked=True, sink=0.0)
    right = GatedLinearHeads(width, int(r["heads"]), int(r["dim"]), int(r.get("vdim") or r["dim"]), int(rank),
                             float(r.get("tau", 1.0)), eps, layer_idx, dtype)
    return ParallelNormed(left, right, width, dtype)


class BapovikLayer(nn.Module):
    def __init__(self, width: int, spec: dict, eps: float, layer_idx: int, dtype: torch.dtype, shapes: Shapes,
                 earlier: List["BapovikLayer"]):
        super().__init__()
        self.norm1 = ResidualRMSNorm(width, eps, dtype)
        kind, m = spec.get("type"), spec["mixer"]
        if kind == "attention":
            source = None
            if m.get("kv_from") is not None:
                j = int(m["kv_from"])
                if not 0 <= j < layer_idx:
                    raise ValueError(f"layer {layer_idx}: kv_from {j} names no earlier layer")
                source = earlier[j].heads
            self.mix = AttentionMixer(width, m, eps, layer_idx, dtype, source)
        elif kind == "parallel":
            self.mix = _parallel(width, m, eps, layer_idx, dtype, shapes)
        else:
            raise ValueError(f"layer {layer_idx}: unknown mixer type {kind!r}")
        mlp = spec.get("mlp")
        self.mlp = None
        if mlp is not None:
            if mlp.get("kind") != "moe":
                raise ValueError(f"layer {layer_idx}: unknown feed-forward kind {mlp.get('kind')!r}")
            self.mlp = PlainTopKMoE(width, int(mlp["expert"]["ff"]), int(mlp["router"]["experts"]),
                                    int(mlp["router"]["top"]), dtype, activation="relu2", scores="sigmoid",
                                    weigh_input=True)

    @property
    def heads(self) -> GatedHeads:
        """The layer's softmax attention (of a parallel mixer: its left half)."""
        return self.mix.left if isinstance(self.mix, ParallelNormed) else self.mix.inner

    def forward(self, x: torch.Tensor, h: torch.Tensor, then: ResidualRMSNorm) -> torch.Tensor:
        """``x``: fp32 residual stream (updated in place), ``h = norm1(x)``; returns ``then(x)`` after this layer.  The
        norms of a parallel mixer's halves, every residual add and the norm that follows are one launch."""
        y = self.mix(h)
        f = self.mlp(h) if self.mlp is not None else None
        if isinstance(self.mix, ParallelNormed):
            return then.after_pair(y[0], self.mix.left_out, y[1], self.mix.right_out, 0.5, f, x)
        return then.add(x, y, f)


class BapovikForCausalLM(nn.Module):
    has_request_state = True          # recurrent halves remember a state per request: no prefix reuse
    residual_dtype = torch.float32

    def __init__(self, vllm_config: VllmConfig):
        super().__init__()
        mc = vllm_config.model_config
        cfg, dtype = mc.hf_config, mc.torch_dtype
        self.cfg, self.dtype = cfg, dtype
        if get_tensor_model_parallel_world_size() > 1 or get_pp_group().world_size > 1:
            raise NotImplementedError("Bapovik runs on one device: its norms reduce over whole rows and its recurrent "
                                      "state is not sharded")
        self.is_first = self.is_last = True
        from ..config import resolve_model_path
        from .loader import checkpoint_tensor_shapes
        shapes = {} if mc.load_format == "dummy" else checkpoint_tensor_shapes(resolve_model_path(mc.model))
        width, eps = int(cfg["width"]), float((cfg.get("norm") or {}).get("eps", 1e-5))
        specs = cfg["layers"]
        if not specs:
            raise ValueError("a Bapovik model needs at least one layer")
        self.width, self.eps, self.vocab = width, eps, int(cfg["vocab"])
        self.start_layer, self.end_layer = 0, len(specs)
        self.embed = VocabParallelEmbedding(self.vocab, width, dtype)
        layers: List[BapovikLayer] = []
        for i, s in enumerate(specs):
            layers.append(BapovikLayer(width, s, eps, i, dtype, shapes, layers))
        self.layers = nn.ModuleList(layers)
        self.final_norm = ResidualRMSNorm(width, eps, dtype)
        self.head = ColumnParallelLinear(width, [self.vocab], False, dtype)
        self.trace_residual: Optional[List[torch.Tensor]] = None      # tests: the residual stream after every layer

    def rebind_buffers(self) -> None:
        return None

    def attention_layers(self) -> List[Attention]:
        """The layers that own keys and values (a layer that reads another's owns none)."""
        return [l.heads.attn for l in self.layers if l.heads.attn.source is None]

    def state_layers(self) -> List[SlotState]:
        return [l.mix.right.slot_state for l in self.layers if isinstance(l.mix, ParallelNormed)]

    def decode_capturable(self) -> bool:
        return all(l.mlp.decode_capturable(self.dtype) for l in self.layers if l.mlp is not None)

    def forward(self, input_ids, positions, intermediate: Optional[IntermediateTensors] = None):
        x = ops.embed_scaled(input_ids, self.embed.weight, 1.0)
        n = len(self.layers)
        h = self.layers[0].norm1(x)
        for i, layer in enumerate(self.layers):
            h = layer(x, h, self.layers[i + 1].norm1 if i + 1 < n else self.final_norm)
            if self.trace_residual is not None:
                self.trace_residual.append(x.clone())
        return h

    def compute_logits(self, hidden: torch.Tensor) -> torch.Tensor:
        return ops.linear_f32(hidden, self.head.weight)[..., :self.vocab]

    # ------------------------------------------------------------ weights
    # leaf -> (parameter under the mixer, what becomes of the tensor: None = the whole parameter, an index = the shard of a
    # bias, (group, index) = a sub-matrix of the fused projection)
    _ATTENTION = {"q": ("proj.weight", (0, 0)), "k": ("proj.weight", (0, 1)), "v": ("proj.weight", (0, 2)),
                  "g": ("proj.weight", (0, -1)), "q.b": ("inner.bias", 0), "k.b": ("inner.bias", 1),
                  "v.b": ("inner.bias", 2), "o": ("o.weight", None)}
    _LEFT = {"q": ("proj.weight", (0, 0)), "k": ("proj.weight", (0, 1)), "v": ("proj.weight", (0, 2)),
             "g": ("proj.weight", (0, 3)), "q.b": ("left.bias", 0), "k.b": ("left.bias", 1), "v.b": ("left.bias", 2),
             "q.norm": ("left.q_norm", None), "k.norm": ("left.k_norm", None), "o": ("left_o.weight", None),
             "out": ("left_out", None)}
    _RIGHT = {"q": ("proj.weight", (1, 0)), "k": ("proj.weight", (1, 1)), "v": ("proj.weight", (1, 2)),
              "g": ("proj.weight", (1, 3)), "a1": ("proj.weight", (1, 4)), "a2": ("right.a2.weight", None),
              "a2.b": ("right.a2_bias", None), "norm": ("right.norm", None), "o": ("right_o.weight", None),
              "out": ("right_out", None)}

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
        if rest == "norm1":
            return base + "norm1.weight", None
        kind, _, leaf = rest.partition(".")
        if kind == "mix":
            if isinstance(layer.mix, ParallelNormed):
                half, _, leaf = leaf.partition(".")
                table = {"left": self._LEFT, "right": self._RIGHT}.get(half, {})
            else:
                table = self._ATTENTION
                if layer.mix.inner.attn.source is not None and leaf[:1] in ("k", "v"):
                    return None
            if leaf not in table:
                return None
            p, shard = table[leaf]
            if isinstance(shard, tuple):
                group, i = shard
                if i < 0:                 # the gate: the group's last sub-matrix
                    i += len(layer.mix.inner.sizes)
                shard = layer.mix.proj.shard(group, i)
            return base + "mix." + p, shard
        if kind != "mlp" or layer.mlp is None:
            return None
        if leaf == "router":
            return base + "mlp.gate.weight", None
        e, _, part = leaf.partition(".")
        if e[:1] == "e" and e[1:].isdigit() and int(e[1:]) < layer.mlp.num_experts and part in ("up", "down"):
            return base + ("mlp.w1" if part == "up" else "mlp.w2"), int(e[1:])
        return None

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
            if loader is not None:
                loader(p, w, shard)
            else:
                w = materialize(w)
                assert w.numel() == p.numel(), (name, tuple(w.shape), tuple(p.shape))
                p.data.copy_(w.reshape(p.shape))
            loaded.append(name)
        return loaded


def weight_shapes(c: dict) -> Shapes:
    """Checkpoint tensor names and shapes of a Bapovik config (for the random-weight loader)."""
    width, vocab = int(c["width"]), int(c["vocab"])
    out: Shapes = {"embed": (vocab, width)}

    def heads_of(q: str, m: dict, own: bool) -> None:
        heads, kvh, dim = int(m["heads"]), int(m.get("kv_heads") or m["heads"]), int(m["dim"])
        vdim = int(m.get("vdim") or dim)
        for nm, rows in (("q", heads * dim),) + ((("k", kvh * dim), ("v", kvh * vdim)) if own else ()):
            out[q + nm], out[q + nm + ".b"] = (rows, width), (rows,)
        out[q + "g"], out[q + "o"] = (heads, width), (width, heads * vdim)

    for i, spec in enumerate(c["layers"]):
        m, p = spec["mixer"], f"l{i}."
        out[p + "norm1"] = (width,)
        if spec["type"] == "parallel":
            q = p + "mix.left."
            heads_of(q, m["left"], True)
            out[q + "q.norm"], out[q + "k.norm"], out[q + "out"] = (int(m["left"]["dim"]),), (int(m["left"]["dim"]),), (width,)
            r, q = m["right"], p + "mix.right."
            heads, dim, vdim, rank = int(r["heads"]), int(r["dim"]), int(r.get("vdim") or r["dim"]), int(r["decay_rank"])
            for nm, rows in (("q", heads * dim), ("k", heads * dim), ("v", heads * vdim), ("g", heads * vdim)):
                out[q + nm] = (rows, width)
            out[q + "o"], out[q + "norm"], out[q + "out"] = (width, heads * vdim), (vdim,), (width,)
            out[q + "a1"], out[q + "a2"], out[q + "a2.b"] = (rank, width), (heads * dim, rank), (heads * dim,)
        elif spec["type"] == "attention":
            heads_of(p + "mix.", m, m.get("kv_from") is None)
        else:
            raise ValueError(f"layer {i}: unknown mixer type {spec['type']!r}")
        mlp = spec.get("mlp")
        if mlp:
            ff, experts = int(mlp["expert"]["ff"]), int(mlp["router"]["experts"])
            for e in range(experts):
                out[f"{p}mlp.e{e}.up"], out[f"{p}mlp.e{e}.down"] = (ff, width), (width, ff)
            out[p + "mlp.router"] = (experts, width)
    out["final.norm"], out["head"] = (width,), (vocab, width)
    return out


def random_weight(name: str, shape: Tuple[int, ...], gen: torch.Generator, device, dtype) -> torch.Tensor:
    """A plausible random value for a checkpoint tensor (projections that keep the variance, gains around one, small
    biases, decays spread over (0, 1))."""
    def uni(lo: float, hi: float) -> torch.Tensor:
        return lo + (hi - lo) * torch.rand(shape, generator=gen, device=device, dtype=torch.float32)
    leaf = name.rsplit(".", 1)[-1]
    if leaf in ("norm1", "norm", "out"):
        w = uni(0.8, 1.2)
    elif name.endswith("a2.b"):
        w = uni(-1.0, 4.0)
    elif leaf == "b":
        w = uni(-0.3, 0.3)
    elif name == "embed":
        w = uni(-1.0, 1.0)
    else:
        s = (3.0 / shape[-1]) ** 0.5
        w = uni(-s, s)
    return w.to(dtype)
