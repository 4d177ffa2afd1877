"""Runidra: a pre-norm decoder whose config lists its layers one by one, like
Vurizen's, Sogidra's, Zabusun's and Pudizen's, with these pieces:

* hyper-connections: `streams` copies of the residual stream; a sublayer reads
  one weighted sum of them and writes back to all of them through a small
  matrix (hyper_connections.HyperConnection, ops.hyper_rmsnorm); all copies
  start as the embedding and the logits read their sum;
* a loop: layers start .. stop - 1 run `times` times in a row with the same
  weights, every pass with a cache entry or recurrent state of its own. The
  config reader unrolls it: this module, the cache geometry and the layer
  ranges of pipeline stages count layer RUNS;
* mixer 'mlstm': matrix LSTM with exponential input gates and soft-capped
  gate pre-activations (linear_attention.MLSTM);
* mixer 'latent_attention': queries through a normed latent, keys and values
  expanded from a cached normed latent, a rotated key part shared by all heads
  (pairs 2i, 2i + 1), sliding window, softmax with a sink per head
  (latent_attention.LatentWindowAttention);
* feed-forward: dense, gelu-gated with biases everywhere, or routed experts
  (softmax over the chosen logits, a logit bias per expert) plus a shared
  expert behind a sigmoid gate (moe.SharedExpertMoE), or none;
* logits: RMS norm, a separate output matrix, times `logit_scale`, through a
  tanh soft cap.

The streams and every norm are fp32 whatever the activation dtype. One kernel
per sublayer writes its result back (dense bias, shared expert's gate and sum
included) and reads and norms the next sublayer's input. Every size and
constant comes from the config or a tensor's shape; layer runs shard by range
(pipeline stages), the fp32 streams travel between stages.

Checkpoint tensor names: 'embed', 'final.norm', 'head', 'l<i>.norm1',
'l<i>.norm2', 'l<i>.hc1.{in,out,mix}', 'l<i>.hc2.{in,out,mix}',
'l<i>.mix.{q,k,v,g,o,norm,i,i.b,f,f.b}' (mlstm),
'l<i>.mix.{dq,dq.norm,uq,dkv,dkv.norm,uk,uv,sink,o}' (latent attention),
'l<i>.mlp.{gate,up,down}[.b]' (dense), 'l<i>.mlp.{router,router.b,
e<j>.{gate,up,down},shared.{gate,up,down,sg}}' (experts).
"""

from __future__ import annotations

import dataclasses
import math
from typing import Callable, List, Optional

import torch
import torch.nn as nn

from .. import ops
from ..parallel.comm import get_comm
from ..parallel.layers import (
    ColumnParallelLinear, MergedColumnParallelLinear, RowParallelLinear,
    VocabEmbedding,
)
from .config import ModelConfig, feed_forward_kind
from .forward_meta import ForwardMeta
from .hyper_connections import HyperConnection
from .latent_attention import LatentWindowAttention
from .linear_attention import MLSTM
from .moe import FusedMoE, SharedExpertMoE
from .registry import register_model


class BiasedGluMLP(nn.Module):
    """W_down (gelu_tanh(W_gate h + b_gate) * (W_up h + b_up)) + b_down. The
    last bias is left to the caller's residual kernel (`down_bias`)."""

    def __init__(self, hidden_size: int, ff: int):
        super().__init__()
        self.gate_up = MergedColumnParallelLinear(hidden_size, [ff, ff])
        self.gate_up_bias = nn.Parameter(torch.empty(2 * ff), requires_grad=False)
        self.down = RowParallelLinear(ff, hidden_size)
        self.down_bias = nn.Parameter(torch.empty(hidden_size), requires_grad=False)
        self.ff = ff

    def forward(self, x: torch.Tensor) -> torch.Tensor:
        return self.down(ops.biased_glu(self.gate_up(x), self.gate_up_bias,
                                        "gelu_tanh"))


def _moe_config(cfg: ModelConfig, mlp: dict) -> ModelConfig:
    """The flat MoE fields of ModelConfig for ONE layer's experts."""
    router = mlp["router"]
    return dataclasses.replace(
        cfg,
        num_experts=int(router["experts"]),
        num_experts_per_tok=int(router["top"]),
        moe_intermediate_size=int(mlp["expert"]["ff"]),
        scoring_func="softmax",
        norm_topk_prob=True,
        n_group=1,
        topk_group=1,
    )


class RunidraLayer(nn.Module):
    """The weights of one layer; its runs differ in their cache entry only."""

    def __init__(self, cfg: ModelConfig, spec: dict):
        super().__init__()
        W, eps = cfg.hidden_size, cfg.rms_norm_eps
        self.kind = spec["type"]
        mx = spec["mixer"]
        if self.kind == "mlstm":
            self.mixer = MLSTM(W, int(mx["heads"]), int(mx["dim"]),
                               int(mx["vdim"]), float(mx["gate_cap"]), eps)
        else:
            rot = mx.get("rot") or {}
            self.mixer = LatentWindowAttention(
                W, int(mx["heads"]), int(mx["dim"]), int(mx["rot_dim"]),
                int(mx["vdim"]), int(mx["kv_rank"]), int(mx["mask"]["size"]),
                float(mx["scale"]), eps, 0, True,
                rot_dims=int(rot.get("dims", mx["rot_dim"])),
                rot_base=float(rot.get("base", 10000.0)),
                q_rank=int(mx["q_rank"]), rot_interleaved=True, sink=True)
        self.norm1 = nn.Parameter(torch.empty(W), requires_grad=False)
        self.hc1 = HyperConnection(cfg.streams)
        self.mlp = None
        mlp = spec.get("mlp")
        if mlp is not None:
            if feed_forward_kind(mlp) == "dense":
                self.mlp = BiasedGluMLP(W, int(mlp["ff"]))
            else:
                self.mlp = SharedExpertMoE(
                    _moe_config(cfg, mlp), int((mlp.get("shared") or {}).get("ff", 0)))
            self.norm2 = nn.Parameter(torch.empty(W), requires_grad=False)
            self.hc2 = HyperConnection(cfg.streams)


@register_model("Runidra")
class RunidraShardModel(nn.Module):
    """Layer runs [start_layer, end_layer) of a Runidra stack. The first shard
    owns the embedding, the last one the final norm and the output matrix.
    Between shards the hidden state is the fp32 streams side by side
    (`hidden_dtype`, `hidden_width`). Runs of one layer on one shard share
    its weights."""

    hidden_dtype = torch.float32

    def __init__(self, cfg: ModelConfig, start_layer: int = 0,
                 end_layer: Optional[int] = None):
        super().__init__()
        if cfg.layer_specs is None or cfg.layer_weights is None:
            raise ValueError("Runidra needs a config with a 'layers' list")
        if get_comm().tp_size != 1:
            raise NotImplementedError(
                "Runidra shards by layer range (pipeline stages); tensor "
                "parallelism inside a layer is not wired up for it")
        self.cfg = cfg
        self.start_layer = start_layer
        self.end_layer = end_layer if end_layer is not None else cfg.num_layers
        self.is_first = start_layer == 0
        self.is_last = self.end_layer == cfg.num_layers
        self.eps = cfg.rms_norm_eps
        W = cfg.hidden_size
        self.hidden_width = cfg.streams * W
        if self.is_first:
            self.embed_tokens = VocabEmbedding(cfg.vocab_size, W)
        # one module per layer that runs here, in the order of first use
        self._local = {}
        layers = []
        # (module, entry among this shard's caches or states) of every run
        self.runs: List[tuple] = []
        n_cache = n_state = 0
        for r in range(self.start_layer, self.end_layer):
            i, spec = cfg.layer_weights[r], cfg.layer_specs[r]
            if i not in self._local:
                self._local[i] = len(layers)
                layers.append(RunidraLayer(cfg, spec))
            if spec["type"] == "mlstm":
                entry, n_state = n_state, n_state + 1
            else:
                entry, n_cache = n_cache, n_cache + 1
            self.runs.append((self._local[i], entry))
        self.layers = nn.ModuleList(layers)
        if self.is_last:
            self.norm = nn.Parameter(torch.empty(W), requires_grad=False)
            self.lm_head = ColumnParallelLinear(W, cfg.vocab_size)
        self._sum = None        # the final read: every stream once
        self.rope_cache = None  # angles are computed inside the kernels
        # debugging aid: called with (index of the layer run, fp32 sum of the
        # streams after it) when set
        self.tap: Optional[Callable[[int, torch.Tensor], None]] = None

    @property
    def graph_safe(self) -> bool:
        """Whether a decode forward can be captured into a hipGraph: the
        per-expert loop that serves expert sizes outside the grouped-GEMM
        kernel's tiling reads routing results on the host."""
        W = self.cfg.hidden_size
        return all(
            not isinstance(layer.mlp, SharedExpertMoE)
            or FusedMoE.grouped_kernel_fits(W, layer.mlp.experts.intermediate_size)
            for layer in self.layers
        )

    @property
    def num_local_layers(self) -> int:
        return len(self.runs)

    def embed(self, input_ids: torch.Tensor) -> torch.Tensor:
        assert self.is_first, "only the first shard embeds tokens"
        return ops.embed_streams(input_ids, self.embed_tokens.weight,
                                 self.cfg.streams)

    def forward(self, hidden: torch.Tensor, meta: ForwardMeta) -> torch.Tensor:
        """hidden [T, streams * width] fp32. Returns the final-normed
        activations on the last shard, the streams elsewhere. A sublayer's
        result waits in `pend` and is written back by the kernel that reads
        the next sublayer's input."""
        x = hidden.float().contiguous()
        dev, eps, S = x.device, self.eps, self.cfg.streams
        if self.is_last:
            dt = self.norm.dtype
        else:
            dt = self.layers[0].norm1.dtype if len(self.layers) else x.dtype
        pend = (None,) * 6   # y, y_bias, y2, gate2, mix, write

        for r, (n, entry) in enumerate(self.runs):
            layer = self.layers[n]
            read, write, mix = layer.hc1.f32(dev)
            h = ops.hyper_rmsnorm(x, *pend, read, layer.norm1, eps, dt)
            if self.tap is not None and r > 0:
                self.tap(self.start_layer + r - 1, self._sum_of(x))
            pend = (layer.mixer(h, meta, entry), None, None, None, mix, write)
            if layer.mlp is not None:
                read, write, mix = layer.hc2.f32(dev)
                h = ops.hyper_rmsnorm(x, *pend, read, layer.norm2, eps, dt)
                if isinstance(layer.mlp, SharedExpertMoE):
                    y, y2, gate2 = layer.mlp(h)
                    pend = (y, None, y2, gate2, mix, write)
                else:
                    pend = (layer.mlp(h), layer.mlp.down_bias, None, None, mix, write)
        if self.is_last:
            if self._sum is None or self._sum.device != dev:
                self._sum = torch.ones(S, dtype=torch.float32, device=dev)
            out = ops.hyper_rmsnorm(x, *pend, self._sum, self.norm, eps, dt)
        else:
            if pend[0] is not None:
                ops.hyper_rmsnorm(x, *pend, None, None, eps, dt)
            out = x
        if self.tap is not None and self.runs:
            self.tap(self.end_layer - 1, self._sum_of(x))
        return out

    def _sum_of(self, x: torch.Tensor) -> torch.Tensor:
        return x.view(x.shape[0], self.cfg.streams, -1).sum(1)

    def compute_logits(self, hidden: torch.Tensor) -> torch.Tensor:
        assert self.is_last, "only the last shard computes logits"
        return ops.softcap_logits(self.lm_head(hidden.contiguous()),
                                  self.cfg.logit_scale, self.cfg.logit_softcap)

    def finalize_weights(self) -> None:
        for layer in self.layers:
            layer.mixer.invalidate_constants()
            layer.hc1.invalidate_constants()
            if layer.mlp is not None:
                layer.hc2.invalidate_constants()
                if isinstance(layer.mlp, SharedExpertMoE):
                    layer.mlp.invalidate_constants()

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
                local = self._local.get(int(first[1:]))
                if local is not None:
                    return f"layers.{local}.{rest}"
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
        layer: RunidraLayer = self.layers[int(parts[1])]
        part, key = parts[2], ".".join(parts[3:])
        if part in ("norm2", "hc2", "mlp") and layer.mlp is None:
            return False  # a layer without feed-forward has no use for them
        if part in ("norm1", "norm2") and not key:
            getattr(layer, part).data.copy_(t)
            return True
        if part in ("hc1", "hc2"):
            name = {"in": "read", "out": "write", "mix": "mix"}.get(key)
            if name is None:
                return False
            getattr(getattr(layer, part), name).data.copy_(t)
            return True
        if part == "mix":
            load = self._load_mlstm if layer.kind == "mlstm" else self._load_latent
            return load(layer.mixer, key, t)
        if part == "mlp":
            if isinstance(layer.mlp, BiasedGluMLP):
                return self._load_dense(layer.mlp, key, t)
            return self._load_moe(layer.mlp, parts[3:], t)
        return False

    @staticmethod
    def _load_mlstm(m: MLSTM, key: str, t: torch.Tensor) -> bool:
        slot = {"q": 0, "k": 1, "v": 2, "g": 3}.get(key)
        if slot is not None:
            m.in_proj.load_full_weight_part(slot, t)
        elif key in ("i", "f"):
            m.load_gate("if".index(key), w=t)
        elif key in ("i.b", "f.b"):
            m.load_gate("if".index(key[0]), b=t)
        elif key == "norm":
            m.norm_weight.data.copy_(t)
        elif key == "o":
            m.o_proj.load_full_weight(t)
        else:
            return False
        return True

    @staticmethod
    def _load_latent(m: LatentWindowAttention, key: str, t: torch.Tensor) -> bool:
        if key == "dq":
            m.in_proj.load_full_weight_part(0, t)
        elif key == "dkv":
            m.in_proj.load_full_weight_part(1, t)
        elif key == "dq.norm":
            m.q_latent_norm.data.copy_(t)
        elif key == "dkv.norm":
            m.latent_norm.data.copy_(t)
        elif key == "uq":
            m.q_up.load_full_weight(t)
        elif key == "uk":
            m.w_uk.data.copy_(t.view(m.heads, m.dn, m.rank))
        elif key == "uv":
            m.w_uv.data.copy_(t.view(m.heads, m.dv, m.rank))
        elif key == "sink":
            m.sink.data.copy_(t)
        elif key == "o":
            m.o_proj.load_full_weight(t)
        else:
            return False
        return True

    @staticmethod
    def _load_dense(m: BiasedGluMLP, key: str, t: torch.Tensor) -> bool:
        if key in ("gate", "up"):
            m.gate_up.load_full_weight_part(0 if key == "gate" else 1, t)
        elif key == "gate.b":
            m.gate_up_bias.data[: m.ff].copy_(t)
        elif key == "up.b":
            m.gate_up_bias.data[m.ff :].copy_(t)
        elif key == "down":
            m.down.load_full_weight(t)
        elif key == "down.b":
            m.down_bias.data.copy_(t)
        else:
            return False
        return True

    @staticmethod
    def _load_moe(m: SharedExpertMoE, parts: List[str], t: torch.Tensor) -> bool:
        router, E = m.experts.router, m.experts.router.num_experts
        if parts == ["router"]:
            router.weight.data[:E].copy_(t)
        elif parts == ["router", "b"]:
            router.logit_bias.data.copy_(t)
        elif len(parts) == 2 and parts[0] == "shared" and m.shared_ff:
            if parts[1] in ("gate", "up"):
                m.gate_up.load_full_weight_part(0 if parts[1] == "gate" else 1, t)
            elif parts[1] == "down":
                m.down.load_full_weight(t)
            elif parts[1] == "sg":
                router.weight.data[E:].copy_(t.view(1, -1))
            else:
                return False
        elif len(parts) == 2 and parts[0][:1] == "e" and parts[0][1:].isdigit():
            e = int(parts[0][1:])
            if parts[1] == "gate":
                m.experts.load_expert_gate(e, t)
            elif parts[1] == "up":
                m.experts.load_expert_up(e, t)
            elif parts[1] == "down":
                m.experts.load_expert_down(e, t)
            else:
                return False
        else:
            return False
        return True

    @torch.no_grad()
    def init_random(self, seed: int = 1234) -> None:
        """Synthetic weights for benchmarking: projections ~ N(0, 1/fan_in),
        norm weights 1, biases and sinks small, forget gates biased towards
        keeping; streams read evenly, kept apart and written alike."""
        g = torch.Generator().manual_seed(seed)
        S = self.cfg.streams
        for name, p in self.named_parameters():
            leaf = name.rsplit(".", 1)[-1]
            if leaf in ("norm", "norm1", "norm2", "norm_weight", "latent_norm",
                        "q_latent_norm"):
                p.data.fill_(1.0)
            elif leaf == "read":
                p.data.fill_(1.0 / S)
            elif leaf == "write":
                p.data.fill_(1.0)
            elif name.endswith((".hc1.mix", ".hc2.mix")):
                p.data.copy_(torch.eye(S))
            elif leaf == "gate_bias":   # [input | forget]
                p.data[: p.numel() // 2].fill_(-2.0)
                p.data[p.numel() // 2 :].fill_(4.0)
            elif leaf in ("sink", "logit_bias", "gate_up_bias", "down_bias"):
                p.data.copy_(torch.randn(p.shape, generator=g).mul_(0.1).to(p.dtype))
            else:
                p.data.copy_(
                    torch.randn(p.shape, generator=g, dtype=torch.float32)
                    .mul_(1.0 / math.sqrt(p.shape[-1])).to(p.dtype))
        self.finalize_weights()
