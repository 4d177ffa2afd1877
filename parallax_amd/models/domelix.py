"""Domelix: a decoder whose config lists its layers one by one, like Vurizen's,
Sogidra's, Zabusun's, Pudizen's and Runidra's, with these pieces:

* a layer has two RMS norms of the SAME stream (weights stored around zero)
  and runs its mixer on one and its feed-forward on the other:
  x += mixer(norm1(x)) + ff(norm2(x));
* mixer 'parallel': softmax attention with a distance bias, sinks and an
  element-wise output gate (row_attention.DistanceBiasAttention) beside
  lightning attention (linear_attention.DecayLinearAttention); both results
  are RMS-normed over the model width and averaged;
* mixer 'delta': gated delta rule behind a short convolution
  (linear_attention.GatedDeltaRule);
* mixer 'retention': rotated queries and keys, a fixed decay per head
  (linear_attention.DecayLinearAttention);
* feed-forward: routed silu-gated experts, softmax scores over all experts,
  optionally limited to the best groups of neighbouring experts (a group is as
  good as its best expert), weights normalised over the chosen; or none;
* logits: RMS norm and an output matrix of their own.

The stream and every norm are fp32 whatever the activation dtype. One kernel
per layer (ops.parallel_rmsnorm_add) norms and averages the two halves of a
'parallel' mixer, adds mixer and feed-forward into the stream and writes both
norms of the next layer. Every size and constant comes from the config or a
tensor's shape; layers shard by range (pipeline stages), the fp32 stream
travels between stages.

Checkpoint tensor names: 'embed', 'final.norm', 'head', 'l<i>.norm1',
'l<i>.norm2', 'l<i>.mix.left.{q,k,v,g,rel,sink,o,out}',
'l<i>.mix.right.{q,k,v,g,norm,o,out}' (parallel),
'l<i>.mix.{q,k,v,g,q.conv,k.conv,v.conv,a,b,A_log,dt_bias,norm,o}' (delta),
'l<i>.mix.{q,k,v,g,o}' (retention),
'l<i>.mlp.{router,e<j>.{gate,up,down}}'.
"""

from __future__ import annotations

import dataclasses
import math
from typing import Callable, List, Optional

import torch
import torch.nn as nn

from .. import ops
from ..parallel.comm import get_comm
from ..parallel.layers import ColumnParallelLinear, VocabEmbedding
from .config import ModelConfig
from .forward_meta import ForwardMeta
from .linear_attention import DecayLinearAttention, GatedDeltaRule
from .moe import FusedMoE, MoERouter
from .parallel_mixer import ParallelMixer
from .registry import register_model
from .row_attention import DistanceBiasAttention


def _moe_config(cfg: ModelConfig, mlp: dict) -> ModelConfig:
    """The flat MoE fields of ModelConfig for ONE layer's experts."""
    router = mlp["router"]
    groups = router.get("groups") or {}
    return dataclasses.replace(
        cfg,
        num_experts=int(router["experts"]),
        num_experts_per_tok=int(router["top"]),
        moe_intermediate_size=int(mlp["expert"]["ff"]),
        scoring_func="softmax",
        norm_topk_prob=True,
        n_group=int(groups.get("count", 1)),
        topk_group=int(groups.get("keep", 1)),
    )


class DomelixLayer(nn.Module):
    # a 'parallel' mixer's result is this times the sum of its normed halves
    half = 0.5

    def __init__(self, cfg: ModelConfig, spec: dict, cache_idx: int, state_idx: int):
        super().__init__()
        W, eps = cfg.hidden_size, cfg.rms_norm_eps
        self.kind = spec["type"]
        mx = spec["mixer"]
        if self.kind == "parallel":
            lf, rt = mx["left"], mx["right"]
            heads = int(lf["heads"])
            left = DistanceBiasAttention(
                W, heads, int(lf.get("kv_heads", heads)), int(lf["dim"]),
                int(lf.get("vdim", lf["dim"])), float(lf["scale"]),
                int(lf["bias_max"]), eps, cache_idx, own_proj=False)
            right = DecayLinearAttention(
                W, int(rt["heads"]), int(rt["dim"]), int(rt.get("vdim", rt["dim"])),
                rt["decay"], eps, state_idx, silu=True, norm_all=True,
                gate_act="sigmoid", own_proj=False)
            self.mixer = ParallelMixer(W, left, right, self.half, self.half)
            self.left_out = nn.Parameter(torch.empty(W), requires_grad=False)
            self.right_out = nn.Parameter(torch.empty(W), requires_grad=False)
        elif self.kind == "delta":
            heads = int(mx["heads"])
            self.mixer = GatedDeltaRule(
                W, heads, int(mx.get("kv_heads", heads)), int(mx["dim"]),
                int(mx.get("vdim", mx["dim"])), int(mx["conv"]), eps, state_idx)
        else:
            rot = mx.get("rot") or {}
            dim = int(mx["dim"])
            self.mixer = DecayLinearAttention(
                W, int(mx["heads"]), dim, int(mx.get("vdim", dim)), mx["decay"],
                eps, state_idx, rot_dims=int(rot.get("dims", 0)),
                rot_base=float(rot.get("base", 10000.0)), k_scale=dim ** -0.5)
        self.norm1 = nn.Parameter(torch.empty(W), requires_grad=False)
        self.mlp = None
        mlp = spec.get("mlp")
        if mlp is not None:
            mc = _moe_config(cfg, mlp)
            self.mlp = FusedMoE(mc, router=MoERouter(mc, fused=True))
            self.mlp.fp32_output = True
            self.norm2 = nn.Parameter(torch.empty(W), requires_grad=False)


@register_model("Domelix")
class DomelixShardModel(nn.Module):
    """Layers [start_layer, end_layer) of a Domelix stack. The first shard owns
    the embedding, the last one the final norm and the output matrix. Between
    shards the hidden state IS the fp32 residual stream (`hidden_dtype`)."""

    hidden_dtype = torch.float32

    def __init__(self, cfg: ModelConfig, start_layer: int = 0,
                 end_layer: Optional[int] = None):
        super().__init__()
        if cfg.layer_specs is None:
            raise ValueError("Domelix needs a config with a 'layers' list")
        if get_comm().tp_size != 1:
            raise NotImplementedError(
                "Domelix shards by layer range (pipeline stages); tensor "
                "parallelism inside a layer is not wired up for it")
        self.cfg = cfg
        self.start_layer = start_layer
        self.end_layer = end_layer if end_layer is not None else cfg.num_layers
        self.is_first = start_layer == 0
        self.is_last = self.end_layer == cfg.num_layers
        self.eps = cfg.rms_norm_eps
        W = cfg.hidden_size
        if self.is_first:
            self.embed_tokens = VocabEmbedding(cfg.vocab_size, W)
        # every layer owns a state entry, a 'parallel' one a cache entry too
        layers, n_cache = [], 0
        for n, g in enumerate(range(self.start_layer, self.end_layer)):
            spec = cfg.layer_specs[g]
            layers.append(DomelixLayer(cfg, spec, n_cache, n))
            n_cache += spec["type"] == "parallel"
        self.layers = nn.ModuleList(layers)
        if self.is_last:
            self.norm = nn.Parameter(torch.empty(W), requires_grad=False)
            self.lm_head = ColumnParallelLinear(W, cfg.vocab_size)
        self.rope_cache = None  # the rotation's table is built per forward
        self._side = None       # the experts' stream
        # debugging aid: called with (global layer index, fp32 residual after
        # that layer) when set
        self.tap: Optional[Callable[[int, torch.Tensor], None]] = None

    @property
    def graph_safe(self) -> bool:
        """Whether a decode forward can be captured into a hipGraph: the
        per-expert loop that serves expert sizes outside the grouped-GEMM
        kernel's tiling reads routing results on the host."""
        W = self.cfg.hidden_size
        return all(
            layer.mlp is None
            or FusedMoE.grouped_kernel_fits(W, layer.mlp.intermediate_size)
            for layer in self.layers
        )

    @property
    def num_local_layers(self) -> int:
        return len(self.layers)

    def embed(self, input_ids: torch.Tensor) -> torch.Tensor:
        assert self.is_first, "only the first shard embeds tokens"
        return self.embed_tokens(input_ids)

    def forward(self, hidden: torch.Tensor, meta: ForwardMeta) -> torch.Tensor:
        """hidden [T, width]: embedding rows (first shard) or the previous
        shard's fp32 residual. Returns the final-normed activations on the
        last shard, the fp32 residual elsewhere. A layer's results wait in
        `pend` and are added by the kernel that writes the next layer's
        norms."""
        x = hidden.float().contiguous()
        dev = x.device
        if self.is_last:
            dt = self.norm.dtype
        else:
            dt = self.layers[0].norm1.dtype if len(self.layers) else x.dtype
        pend = (None, None, None, None, 1.0, None)   # a, b, wa, wb, scale, f
        # Mixer and feed-forward do not read each other, so the experts (grouped
        # GEMMs) run on a stream of their own beside the mixer, whose recurrent
        # kernels leave most of the chip idle; in a captured decode step they
        # are two branches of the graph. Every tensor that crosses is waited
        # for before its owner lets go of it: h2 and f live until the streams
        # have joined, and the next layer's fork waits for the kernel that
        # read f.
        main = side = None
        if x.is_cuda and dt == torch.bfloat16 and self.graph_safe:
            main = torch.cuda.current_stream(dev)
            if self._side is None:
                self._side = torch.cuda.Stream(dev)
            side = self._side

        for i, layer in enumerate(self.layers):
            w2 = layer.norm2 if layer.mlp is not None else None
            h1, h2 = ops.parallel_rmsnorm_add(x, *pend, layer.norm1, w2, self.eps,
                                              1.0, dt)
            if self.tap is not None and i > 0:
                self.tap(self.start_layer + i - 1, x)
            f = None
            if layer.mlp is not None and side is not None:
                side.wait_stream(main)
                with torch.cuda.stream(side):
                    f = layer.mlp(h2)
            if layer.kind == "parallel":
                a, b = layer.mixer(h1, meta)
                pend = (a, b, layer.left_out, layer.right_out, layer.half)
            else:
                pend = (layer.mixer(h1, meta), None, None, None, 1.0)
            if layer.mlp is not None:
                if side is not None:
                    main.wait_stream(side)
                else:
                    f = layer.mlp(h2)
            pend += (f,)
        w = self.norm if self.is_last else None
        out = x
        if w is not None or pend[0] is not None:
            h, _ = ops.parallel_rmsnorm_add(x, *pend, w, None, self.eps, 1.0, dt)
            out = h if self.is_last else x
        if self.tap is not None and len(self.layers):
            self.tap(self.end_layer - 1, x)
        return out

    def compute_logits(self, hidden: torch.Tensor) -> torch.Tensor:
        assert self.is_last, "only the last shard computes logits"
        return self.lm_head(hidden.contiguous()).float()

    def finalize_weights(self) -> None:
        for layer in self.layers:
            layer.mixer.invalidate_constants()

    # -- weight loading ---------------------------------------------------------

    def map_global_layer(self, name: str) -> Optional[str]:
        """Checkpoint name -> 'layers.<local>.<rest>' or the name itself when
        this shard holds the tensor, else None."""
        if name == "embed":
            return name if self.is_first else None
        if name in ("final.norm", "head"):
            return name if self.is_last else None
        if name.startswith("l"):
            first, _, rest = name.partition(".")
            if first[1:].isdigit() and rest:
                g = int(first[1:])
                if self.start_layer <= g < self.end_layer:
                    return f"layers.{g - self.start_layer}.{rest}"
        return None

    def load_hf_weight(self, name: str, tensor: torch.Tensor) -> bool:
        local = self.map_global_layer(name)
        if local is None:
            return False
        t = tensor.to(torch.bfloat16) if tensor.is_floating_point() else tensor
        if local == "embed":
            self.embed_tokens.weight.data.copy_(t)
            return True
        if local == "final.norm":
            self.norm.data.copy_(t)
            return True
        if local == "head":
            self.lm_head.load_full_weight(t)
            return True
        parts = local.split(".")
        layer: DomelixLayer = self.layers[int(parts[1])]
        part, key = parts[2], ".".join(parts[3:])
        if part in ("norm2", "mlp") and layer.mlp is None:
            return False  # a layer without feed-forward has no use for them
        if part in ("norm1", "norm2") and not key:
            getattr(layer, part).data.copy_(t)
            return True
        if part == "mix":
            if layer.kind == "parallel" and len(parts) > 4:
                return self._load_half(layer, parts[3], ".".join(parts[4:]), t)
            if layer.kind == "delta":
                return self._load_delta(layer.mixer, key, t)
            if layer.kind == "retention":
                return self._load_decay(layer.mixer, layer.mixer.in_proj, 0, key, t)
        if part == "mlp":
            return self._load_moe(layer.mlp, parts[3:], t)
        return False

    def _load_half(self, layer: DomelixLayer, side: str, key: str,
                   t: torch.Tensor) -> bool:
        mixer: ParallelMixer = layer.mixer
        if key == "out" and side in ("left", "right"):
            (layer.left_out if side == "left" else layer.right_out).data.copy_(t)
            return True
        if side == "right":
            return self._load_decay(mixer.right, mixer.in_proj, mixer.n_left, key, t)
        if side != "left":
            return False
        m: DistanceBiasAttention = mixer.left
        slot = {"q": 0, "k": 1, "v": 2, "g": 3}.get(key)
        if slot is not None:
            mixer.in_proj.load_full_weight_part(slot, t)
        elif key == "rel":
            m.load_rel(t)
        elif key == "sink":
            m.sink.data.copy_(t)
        elif key == "o":
            m.o_proj.load_full_weight(t)
        else:
            return False
        return True

    @staticmethod
    def _load_decay(m: DecayLinearAttention, in_proj, first: int, key: str,
                    t: torch.Tensor) -> bool:
        """first: the part of in_proj where this mixer's projections start."""
        slot = {"q": 0, "k": 1, "v": 2, "g": 3}.get(key)
        if slot is not None:
            in_proj.load_full_weight_part(first + slot, t)
        elif key == "norm" and m.norm_weight is not None:
            m.norm_weight.data.copy_(t)
        elif key == "o":
            m.o_proj.load_full_weight(t)
        else:
            return False
        return True

    @staticmethod
    def _load_delta(m: GatedDeltaRule, key: str, t: torch.Tensor) -> bool:
        slot = {"q": 0, "k": 1, "v": 2, "g": 3}.get(key)
        if slot is not None:
            m.in_proj.load_full_weight_part(slot, t)
        elif key in ("q.conv", "k.conv", "v.conv"):
            m.load_conv("qkv".index(key[0]), t)
        elif key in ("a", "b"):
            m.load_gate("ba".index(key), t)
        elif key == "A_log":
            m.a_log.data.copy_(t)
        elif key == "dt_bias":
            m.dt_bias.data.copy_(t)
        elif key == "norm":
            m.norm_weight.data.copy_(t)
        elif key == "o":
            m.o_proj.load_full_weight(t)
        else:
            return False
        return True

    @staticmethod
    def _load_moe(m: FusedMoE, parts: List[str], t: torch.Tensor) -> bool:
        if parts == ["router"]:
            m.router.weight.data.copy_(t)
        elif len(parts) == 2 and parts[0][:1] == "e" and parts[0][1:].isdigit():
            e = int(parts[0][1:])
            if parts[1] == "gate":
                m.load_expert_gate(e, t)
            elif parts[1] == "up":
                m.load_expert_up(e, t)
            elif parts[1] == "down":
                m.load_expert_down(e, t)
            else:
                return False
        else:
            return False
        return True

    @torch.no_grad()
    def init_random(self, seed: int = 1234) -> None:
        """Synthetic weights for benchmarking: projections ~ N(0, 1/fan_in),
        plain norm weights 1, weights stored around zero 0, distance biases
        and sinks small, delta decays slow."""
        g = torch.Generator().manual_seed(seed)
        for name, p in self.named_parameters():
            leaf = name.rsplit(".", 1)[-1]
            if leaf in ("norm", "norm1", "norm2"):
                p.data.zero_()
            elif leaf in ("left_out", "right_out", "norm_weight"):
                p.data.fill_(1.0)
            elif leaf in ("a_log", "dt_bias"):
                p.data.fill_(-1.0)
            elif leaf in ("rel", "sink"):
                p.data.copy_(torch.randn(p.shape, generator=g).mul_(0.1).to(p.dtype))
            else:
                p.data.copy_(
                    torch.randn(p.shape, generator=g, dtype=torch.float32)
                    .mul_(1.0 / math.sqrt(p.shape[-1])).to(p.dtype))
        self.finalize_weights()
