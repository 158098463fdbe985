"""Sufavik: a decoder-only design with several copies of the stream.

The copies all start as the token's embedding. Every sublayer reads the RMS
norm of a weighted sum of the copies, and its result goes back to every
copy while the copies are mixed by a small matrix. The mixer is an
attention over cached low-rank latents (``latent_attention``: queries
through a normed latent of their own, one shared rotated key part with
blended frequencies, a sigmoid gate per head; a layer may read an earlier
layer's latents instead of projecting its own) or a matrix memory with
exponential gates (``mlstm``). The feed-forward is squared-relu, or routed
silu-gated experts of which some are the identity, next to a gated shared
expert, or absent. The copies are summed before the final norm and the
head.

This module only ASSEMBLES the design from the reusable blocks in
``models/mixers.py``: it parses ``config.json``, declares what cache and
state every layer needs, and maps checkpoint tensor names onto the merged
parameters. The engine's block manager, state-slot manager, scheduler and
sampler serve it like any other model.
"""

from __future__ import annotations

import dataclasses
from typing import Dict, Iterable, List, Optional, Tuple, Union

import torch
import torch.nn as nn

from fusioninfer_amd.config import ModelConfig
from fusioninfer_amd.distributed import parallel_state as ps
from fusioninfer_amd.distributed.layers import ReplicatedLinear
from fusioninfer_amd.models.mixers import (
    GatedMemoryConfig,
    GatedMemoryMixer,
    GatedMLP,
    HyperLayer,
    LatentAttention,
    LatentAttentionConfig,
    RoutedExperts,
    SharedExpertMoE,
    SquaredReluMLP,
)
from fusioninfer_amd.ops import seqmix

ARCHITECTURE = "Sufavik"


@dataclasses.dataclass
class FeedForwardConfig:
    kind: str                       # dense | moe
    ff: int                         # dense: hidden size; moe: per expert
    experts: int = 0
    identity: int = 0               # router outputs after the experts'
    top: int = 0
    shared_ff: int = 0              # 0: no shared expert


@dataclasses.dataclass
class SufavikLayerConfig:
    kind: str                       # latent_attention | mlstm
    mixer: Union[LatentAttentionConfig, GatedMemoryConfig]
    kv_from: Optional[int]          # layer whose latents this one reads
    mlp: Optional[FeedForwardConfig]


@dataclasses.dataclass
class SufavikConfig:
    width: int
    vocab: int
    eps: float
    streams: int
    layers: List[SufavikLayerConfig]


def _parse_mlp(i: int, mlp: Optional[dict]) -> Optional[FeedForwardConfig]:
    if not mlp:
        return None
    kind = mlp.get("kind")
    if kind == "dense":
        return FeedForwardConfig("dense", int(mlp["ff"]))
    if kind == "moe":
        r = mlp["router"]
        shared = mlp.get("shared") or {}
        return FeedForwardConfig(
            "moe", int(mlp["expert"]["ff"]), experts=int(r["experts"]),
            identity=int(r.get("identity") or 0), top=int(r["top"]),
            shared_ff=int(shared.get("ff", 0)))
    raise ValueError(f"layer {i}: unknown mlp kind {kind!r}")


def _parse_latent(m: dict) -> LatentAttentionConfig:
    rot = m["rot"]
    sc = rot.get("scaling") or {}
    return LatentAttentionConfig(
        heads=int(m["heads"]), dim=int(m["dim"]), rot_dim=int(m["rot_dim"]),
        vdim=int(m["vdim"]), rank=int(m["kv_rank"]),
        scale=float(m["scale"]), rot_base=float(rot["base"]), sink=False,
        rot_dims=int(rot.get("dims", m["rot_dim"])),
        q_rank=int(m["q_rank"]), head_gate=True,
        rot_factor=float(sc.get("factor", 1.0)),
        rot_original=float(sc.get("original", 0.0)),
        rot_fast=float(sc.get("fast", 0.0)),
        rot_slow=float(sc.get("slow", 0.0)))


def _cached_form(c: LatentAttentionConfig) -> tuple:
    """What two layers must share to read the same cached rows."""
    return (c.rank, c.rot_dim, c.rot_dims, c.rot_base, c.rot_factor,
            c.rot_original, c.rot_fast, c.rot_slow)


def parse_config(raw: dict) -> SufavikConfig:
    """config.json -> SufavikConfig; every size and constant is read from
    the config."""
    layers: List[SufavikLayerConfig] = []
    for i, L in enumerate(raw["layers"]):
        kind, m = L.get("type"), L["mixer"]
        src = None
        if kind == "latent_attention":
            mixer = _parse_latent(m)
            src = m.get("kv_from")
            if src is not None:
                src = int(src)
                if (not 0 <= src < i
                        or layers[src].kind != "latent_attention"
                        or layers[src].kv_from is not None):
                    raise ValueError(
                        f"layer {i}: kv_from {src} must name an earlier "
                        "latent layer with a down projection of its own")
                if _cached_form(layers[src].mixer) != _cached_form(mixer):
                    raise ValueError(
                        f"layer {i}: latent sizes or rotation differ from "
                        f"layer {src}'s")
        elif kind == "mlstm":
            mixer = GatedMemoryConfig(
                heads=int(m["heads"]), dim=int(m["dim"]),
                vdim=int(m["vdim"]), gate_cap=float(m["gate_cap"]))
        else:
            raise ValueError(f"layer {i}: unknown mixer type {kind!r}")
        layers.append(SufavikLayerConfig(kind, mixer, src,
                                         _parse_mlp(i, L.get("mlp"))))
    streams = int(raw["streams"])
    if streams < 1:
        raise ValueError("streams must be at least 1")
    return SufavikConfig(
        width=int(raw["width"]), vocab=int(raw["vocab"]),
        eps=float(raw["norm"]["eps"]), streams=streams, layers=layers)


def model_config_from_dict(raw: dict, model_path: Optional[str] = None,
                           name: str = ARCHITECTURE) -> ModelConfig:
    """Engine-level ModelConfig for a Sufavik config dict (the registry's
    architecture hook)."""
    arch = parse_config(raw)
    first = arch.layers[0].mixer
    if isinstance(first, LatentAttentionConfig):
        kv_heads, dim = 1, first.rank + first.rot_dim
    else:
        kv_heads, dim = first.heads, first.dim
    ffs = [L.mlp for L in arch.layers if L.mlp is not None]
    return ModelConfig(
        name=name,
        architecture=ARCHITECTURE,
        arch=arch,
        hidden_size=arch.width,
        num_layers=len(arch.layers),
        num_heads=first.heads,
        num_kv_heads=kv_heads,
        head_dim=dim,
        intermediate_size=max((f.ff for f in ffs), default=0),
        vocab_size=arch.vocab,
        rms_norm_eps=arch.eps,
        qk_norm=False,
        model_path=model_path,
        max_position_embeddings=1 << 24,
    )


class SufavikLM(nn.Module):
    """embedding -> layers on several copies of the stream -> sum -> final
    RMS norm -> head.

    Engine interface (same as CausalLM): ``forward(ids, meta, caches)``
    returns the final-normed hidden rows, ``compute_logits`` applies the
    head. ``allocate_caches`` hands out one dict per layer (a borrowing
    layer gets the dict of the layer it reads) and ``uses_state_slots``
    makes the runner build sequence-grouped metadata and the scheduler hand
    out state slots."""

    uses_state_slots = True
    supports_prefix_caching = False   # the memory has no block form

    def __init__(self, cfg: ModelConfig):
        super().__init__()
        assert ps.tp_world_size() == 1 and ps.pp_world_size() == 1, (
            "Sufavik runs single-rank (TP/PP sharding of its mixers is "
            "not implemented)")
        self.cfg = cfg
        arch: SufavikConfig = cfg.arch
        self.arch = arch
        dtype = {"bfloat16": torch.bfloat16,
                 "float32": torch.float32}[cfg.dtype]
        self.dtype = dtype
        self.pp_first = self.pp_last = True
        W = arch.width
        base_seed = torch.initial_seed() % (2**62)
        torch.manual_seed(base_seed + 1000003)
        self.embed_tokens = nn.Parameter(
            torch.empty(arch.vocab, W, dtype=dtype).normal_(0.0, 0.02),
            requires_grad=False)
        layers = []
        for i, L in enumerate(arch.layers):
            torch.manual_seed(base_seed + 1000003 * (i + 2))
            if L.kind == "latent_attention":
                mixer = LatentAttention(L.mixer, W, arch.eps, dtype,
                                        own_kv=L.kv_from is None)
            else:
                mixer = GatedMemoryMixer(L.mixer, W, arch.eps, dtype)
            mlp = None
            if L.mlp is not None and L.mlp.kind == "dense":
                mlp = SquaredReluMLP(W, L.mlp.ff, dtype)
            elif L.mlp is not None:
                f = L.mlp
                shared = (GatedMLP(W, f.shared_ff, dtype, act="silu")
                          if f.shared_ff else None)
                mlp = SharedExpertMoE(
                    RoutedExperts(W, f.ff, f.experts, f.top, dtype,
                                  score="softmax", renorm=False,
                                  act="silu_gate", identity=f.identity,
                                  side_gates=1 if f.shared_ff else 0),
                    shared)
            layers.append(HyperLayer(mixer, mlp, arch.streams, W, arch.eps,
                                     dtype))
        self.layers = nn.ModuleList(layers)
        self.final_norm = nn.Parameter(torch.ones(W, dtype=torch.float32),
                                       requires_grad=False)
        self.register_buffer(
            "sum_in", torch.ones(arch.streams, dtype=torch.float32),
            persistent=False)
        torch.manual_seed(base_seed + 1000003 * (len(arch.layers) + 2))
        self.lm_head = ReplicatedLinear(W, arch.vocab, dtype=dtype)
        torch.manual_seed(base_seed + 777)
        # when set to a list, forward appends the sum of the copies after
        # every layer (debugging, layer-by-layer tests)
        self.residual_trace: Optional[list] = None

    # ------------------------------------------------------ engine hooks
    @property
    def num_local_layers(self) -> int:
        return len(self.layers)

    def kv_block_bytes(self, block_size: int) -> int:
        return max(sum(layer.mixer.block_bytes(block_size)
                       for layer in self.layers), 1)

    def allocate_caches(self, num_blocks: int, block_size: int,
                        num_slots: int, device) -> list:
        """One dict per layer: the paged latent rows of its attention (or
        the dict of the layer it borrows from), or the fp32 slot states of
        its memory."""
        caches: list = []
        for layer, L in zip(self.layers, self.arch.layers):
            if L.kv_from is not None:
                caches.append(caches[L.kv_from])
            else:
                caches.append(layer.mixer.state_tensors(
                    num_blocks, block_size, num_slots, device))
        return caches

    # ----------------------------------------------------------- forward
    def forward(self, input_ids, meta, caches, hidden=None, residual=None):
        first = self.layers[0]
        xs, h = seqmix.hyper_start(input_ids, self.embed_tokens,
                                   first.hc1_in, first.norm1, self.arch.eps,
                                   self.dtype)
        n = len(self.layers)
        for i, (layer, cache) in enumerate(zip(self.layers, caches)):
            nxt = ((self.sum_in, self.final_norm) if i + 1 == n else
                   (self.layers[i + 1].hc1_in, self.layers[i + 1].norm1))
            h = layer(xs, h, meta, cache, nxt)
            if self.residual_trace is not None:
                self.residual_trace.append(xs.sum(1))
        return h

    def compute_logits(self, hidden: torch.Tensor) -> torch.Tensor:
        return self.lm_head(hidden).float()

    # ----------------------------------------------------------- weights
    def load_weights(self, tensors: Iterable[Tuple[str, torch.Tensor]]) -> int:
        """Checkpoint names -> parameters. A mixer's input branches land in
        its layer's merged projection, expert matrices in the stacked expert
        tensors, gate and up of the shared expert in one merged matrix, the
        router and the shared expert's scalar gate in one fp32 matrix; norm
        weights, stream vectors and matrices, gate biases and the router
        correction are kept in fp32."""
        n = 0
        seen = set()
        for name, t in tensors:
            self._load_one(name, t)
            seen.add(name)
            n += 1
        missing = [k for k in self.expected_tensor_names() if k not in seen]
        if missing:
            raise ValueError(f"checkpoint lacks tensors: {missing[:8]}"
                             f"{' ...' if len(missing) > 8 else ''}")
        for layer in self.layers:
            if isinstance(layer.mlp, SharedExpertMoE):
                layer.mlp.routed.invalidate_packed()
            if isinstance(layer.mixer, LatentAttention):
                layer.mixer.invalidate_packed()
        return n

    def expected_tensor_names(self) -> List[str]:
        return list(self._name_map())

    def _name_map(self) -> Dict[str, tuple]:
        """checkpoint name -> (parameter, view spec or None)."""
        out: Dict[str, tuple] = {
            "embed": (self.embed_tokens, None),
            "head": (self.lm_head.weight, None),
            "final.norm": (self.final_norm, None),
        }
        for i, layer in enumerate(self.layers):
            p = f"l{i}."
            mp = p + "mix."
            mod = layer.mixer
            for q in (1, 2) if layer.mlp is not None else (1,):
                out[f"{p}norm{q}"] = (getattr(layer, f"norm{q}"), None)
                for part in ("in", "out", "mix"):
                    out[f"{p}hc{q}.{part}"] = (
                        getattr(layer, f"hc{q}_{part}"), None)
            for br in mod.in_names:
                out[mp + br] = (layer.in_proj.weight, layer.in_proj_rows(br))
            out[mp + "o"] = (mod.o_proj.weight, None)
            if isinstance(mod, LatentAttention):
                out[mp + "dq.norm"] = (mod.q_norm, None)
                out[mp + "uq"] = (mod.uq.weight, None)
                if mod.own_kv:
                    out[mp + "dkv.norm"] = (mod.c_norm, None)
                out[mp + "uk"] = (mod.uk, None)
                out[mp + "uv"] = (mod.uv_t, ("heads_t",))
            else:
                out[mp + "i.b"] = (mod.i_bias, None)
                out[mp + "f.b"] = (mod.f_bias, None)
                out[mp + "norm"] = (mod.norm_w, None)
            fp = p + "mlp."
            mlp = layer.mlp
            if isinstance(mlp, SharedExpertMoE):
                r = mlp.routed
                out[fp + "router"] = (r.router, (0, r.outputs))
                out[fp + "correction"] = (r.correction, None)
                for e in range(r.experts):
                    out[f"{fp}e{e}.gate"] = (r.gate_up, ("idx", e, 0, r.ff))
                    out[f"{fp}e{e}.up"] = (r.gate_up, ("idx", e, r.ff, r.ff))
                    out[f"{fp}e{e}.down"] = (r.down, ("idx", e))
                if mlp.shared is not None:
                    s = mlp.shared
                    w = s.gate_up_proj.weight
                    out[fp + "shared.gate"] = (w, (0, s.ff))
                    out[fp + "shared.up"] = (w, (s.ff, s.ff))
                    out[fp + "shared.down"] = (s.down_proj.weight, None)
                    out[fp + "shared.sg"] = (r.router, (r.outputs, 1))
            elif mlp is not None:
                out[fp + "up"] = (mlp.up_proj.weight, None)
                out[fp + "down"] = (mlp.down_proj.weight, None)
        return out

    @staticmethod
    def _view(param, spec):
        dst = param.data
        if spec is None:
            return dst
        if spec[0] == "heads_t":     # stored [H, in, out] per head
            return dst.transpose(1, 2)
        if spec[0] == "idx":
            dst = dst[spec[1]]
            return dst if len(spec) == 2 else dst[spec[2]: spec[2] + spec[3]]
        return dst[spec[0]: spec[0] + spec[1]]

    def _load_one(self, name: str, t: torch.Tensor) -> None:
        names = getattr(self, "_names", None)
        if names is None:
            names = self._names = self._name_map()
        if name not in names:
            raise ValueError(f"unknown tensor {name!r}")
        param, spec = names[name]
        dst = self._view(param, spec)
        if spec is not None and spec[0] == "heads_t" and \
                t.shape == (dst.shape[0] * dst.shape[1], dst.shape[2]):
            t = t.view(dst.shape)
        if dst.shape != t.shape:
            raise ValueError(f"{name}: shape {tuple(t.shape)} does not fit "
                             f"{tuple(dst.shape)}")
        dst.copy_(t.to(dst.dtype))

    def export_weights(self) -> Dict[str, torch.Tensor]:
        """Inverse of load_weights (checkpoint naming), for writing
        random-init models to disk."""
        out = {}
        for k, (p, spec) in self._name_map().items():
            t = self._view(p, spec).detach().clone().contiguous()
            if spec is not None and spec[0] == "heads_t":
                t = t.view(-1, t.shape[-1])
            out[k] = t
        return out

    def randomize_small_params(self, seed: int = 0) -> None:
        """Random-init use (benchmarks, tests): give norm weights, stream
        vectors and matrices, gate biases and corrections non-trivial values
        so every branch contributes."""
        g = torch.Generator().manual_seed(seed)

        def rnd(p, lo, hi):
            p.data.copy_((torch.rand(p.shape, generator=g) * (hi - lo) + lo)
                         .to(device=p.device, dtype=p.dtype))

        rnd(self.final_norm, 0.8, 1.2)
        n = self.arch.streams
        for layer in self.layers:
            mod = layer.mixer
            for q in (1, 2) if layer.mlp is not None else (1,):
                rnd(getattr(layer, f"norm{q}"), 0.5, 1.5)
                rnd(getattr(layer, f"hc{q}_in"), 0.2, 1.0)
                rnd(getattr(layer, f"hc{q}_out"), 0.3, 1.2)
                mix = getattr(layer, f"hc{q}_mix")
                rnd(mix, -0.2, 0.3)
                mix.data += 0.7 * torch.eye(n, device=mix.device)
            if isinstance(mod, LatentAttention):
                rnd(mod.q_norm, 0.5, 1.5)
                if mod.own_kv:
                    rnd(mod.c_norm, 0.5, 1.5)
            else:
                rnd(mod.norm_w, 0.5, 1.5)
                rnd(mod.i_bias, -1.0, 1.0)
                rnd(mod.f_bias, 1.0, 4.0)
            if isinstance(layer.mlp, SharedExpertMoE):
                rnd(layer.mlp.routed.router, -0.5, 0.5)
                rnd(layer.mlp.routed.correction, -0.1, 0.1)
