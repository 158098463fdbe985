"""Vatunex: a decoder-only design with a norm on both sides of a sublayer.

Every sublayer reads the RMS norm of the stream and adds the RMS norm of
its result; the norms' weights are stored as their distance from one. The
mixer is windowed attention over cached low-rank latents
(``latent_attention``: queries through a normed latent of their own, one
shared rotated key part), grouped-query attention (``attention``:
projection biases, normed heads, partial half-rotation with frequencies
stretched for long contexts, a 1 in the softmax denominator, values blended
with those of the first such layer) or a selective state-space recurrence
behind a short convolution (``mamba1``). The feed-forward is a plain GELU
unit, or absent.

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
    LatentAttention,
    LatentAttentionConfig,
    NormedHeadAttention,
    NormedHeadAttentionConfig,
    PlainMLP,
    SandwichNormLayer,
    SelectiveScanConfig,
    SelectiveScanMixer,
)
from fusioninfer_amd.ops import seqmix

ARCHITECTURE = "Vatunex"


@dataclasses.dataclass
class VatunexLayerConfig:
    kind: str                       # latent_attention | attention | mamba1
    mixer: Union[LatentAttentionConfig, NormedHeadAttentionConfig,
                 SelectiveScanConfig]
    ff: int                         # hidden size of the feed-forward, 0: none


@dataclasses.dataclass
class VatunexConfig:
    width: int
    vocab: int
    eps: float
    layers: List[VatunexLayerConfig]


def _window(m: dict) -> int:
    return int((m.get("mask") or {}).get("size") or 0)


def _parse_latent(m: dict) -> LatentAttentionConfig:
    rot = m["rot"]
    return LatentAttentionConfig(
        heads=int(m["heads"]), dim=int(m["dim"]), rot_dim=int(m["rot_dim"]),
        vdim=int(m["vdim"]), rank=int(m["kv_rank"]),
        scale=float(m["scale"]), rot_base=float(rot["base"]), sink=False,
        rot_dims=int(rot.get("dims", m["rot_dim"])),
        q_rank=int(m["q_rank"]), rot_half=True, window=_window(m))


def _parse_attention(m: dict) -> NormedHeadAttentionConfig:
    rot = m.get("rot") or {}
    sc = rot.get("scaling") or {}
    return NormedHeadAttentionConfig(
        heads=int(m["heads"]), kv_heads=int(m.get("kv_heads", m["heads"])),
        dim=int(m["dim"]), vdim=int(m.get("vdim", m["dim"])),
        scale=float(m["scale"]),
        rot_dims=int(rot.get("dims", m["dim"])) if rot else 0,
        rot_base=float(rot.get("base", 10000.0)),
        rot_factor=float(sc.get("factor", 1.0)),
        rot_low=float(sc.get("low", 1.0)),
        rot_high=float(sc.get("high", 1.0)),
        rot_original=float(sc.get("original", 0.0)),
        window=_window(m), one_in_denominator=True,
        v_mix=bool(m.get("v_mix", False)))


def parse_config(raw: dict) -> VatunexConfig:
    """config.json -> VatunexConfig; every size and constant is read from
    the config."""
    layers: List[VatunexLayerConfig] = []
    first_mix = None
    for i, L in enumerate(raw["layers"]):
        kind, m = L.get("type"), L["mixer"]
        if kind == "latent_attention":
            mixer = _parse_latent(m)
        elif kind == "attention":
            mixer = _parse_attention(m)
            if mixer.v_mix:
                size = mixer.kv_heads * mixer.vdim
                first_mix = first_mix or (i, size)
                if size != first_mix[1]:
                    raise ValueError(
                        f"layer {i}: value size {size} differs from layer "
                        f"{first_mix[0]}'s, whose values it blends in")
        elif kind == "mamba1":
            mixer = SelectiveScanConfig(
                inner=int(m["inner"]), state=int(m["state"]),
                dt_rank=int(m["dt_rank"]), conv=int(m["conv"]))
        else:
            raise ValueError(f"layer {i}: unknown mixer type {kind!r}")
        mlp = L.get("mlp")
        if mlp and mlp.get("kind") != "dense":
            raise ValueError(f"layer {i}: unknown mlp kind "
                             f"{mlp.get('kind')!r}")
        layers.append(VatunexLayerConfig(kind, mixer,
                                         int(mlp["ff"]) if mlp else 0))
    if not layers:
        raise ValueError("a model needs at least one layer")
    return VatunexConfig(
        width=int(raw["width"]), vocab=int(raw["vocab"]),
        eps=float(raw["norm"]["eps"]), layers=layers)


def model_config_from_dict(raw: dict, model_path: Optional[str] = None,
                           name: str = ARCHITECTURE) -> ModelConfig:
    """Engine-level ModelConfig for a Vatunex config dict (the registry's
    architecture hook)."""
    arch = parse_config(raw)
    heads = kv_heads = dim = 1     # of the first layer that has heads
    for L in arch.layers:
        if isinstance(L.mixer, LatentAttentionConfig):
            heads, kv_heads = L.mixer.heads, 1
            dim = L.mixer.rank + L.mixer.rot_dim
            break
        if isinstance(L.mixer, NormedHeadAttentionConfig):
            heads, kv_heads = L.mixer.heads, L.mixer.kv_heads
            dim = L.mixer.dim
            break
    return ModelConfig(
        name=name,
        architecture=ARCHITECTURE,
        arch=arch,
        hidden_size=arch.width,
        num_layers=len(arch.layers),
        num_heads=heads,
        num_kv_heads=kv_heads,
        head_dim=dim,
        intermediate_size=max(L.ff for L in arch.layers),
        vocab_size=arch.vocab,
        rms_norm_eps=arch.eps,
        qk_norm=False,
        model_path=model_path,
        max_position_embeddings=1 << 24,
    )


class VatunexLM(nn.Module):
    """embedding -> layers with a norm on both sides of every sublayer ->
    final RMS norm -> head.

    Engine interface (same as CausalLM): ``forward(ids, meta, caches)``
    returns the final-normed hidden rows, ``compute_logits`` applies the
    head. ``allocate_caches`` hands out one dict per layer and
    ``uses_state_slots`` makes the runner build sequence-grouped metadata
    and the scheduler hand out state slots."""

    uses_state_slots = True
    supports_prefix_caching = False   # the recurrence has no block form

    def __init__(self, cfg: ModelConfig):
        super().__init__()
        assert ps.tp_world_size() == 1 and ps.pp_world_size() == 1, (
            "Vatunex runs single-rank (TP/PP sharding of its mixers is "
            "not implemented)")
        self.cfg = cfg
        arch: VatunexConfig = cfg.arch
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
            block = {"latent_attention": LatentAttention,
                     "attention": NormedHeadAttention,
                     "mamba1": SelectiveScanMixer}[L.kind]
            mlp = PlainMLP(W, L.ff, dtype, act="gelu_tanh") if L.ff else None
            layers.append(SandwichNormLayer(
                block(L.mixer, W, arch.eps, dtype), mlp, W, arch.eps, dtype))
        self.layers = nn.ModuleList(layers)
        self.final_norm = nn.Parameter(torch.ones(W, dtype=torch.float32),
                                       requires_grad=False)
        self.register_buffer("one", torch.ones(1, dtype=torch.float32),
                             persistent=False)
        torch.manual_seed(base_seed + 1000003 * (len(arch.layers) + 2))
        self.lm_head = ReplicatedLinear(W, arch.vocab, dtype=dtype)
        torch.manual_seed(base_seed + 777)
        # when set to a list, forward appends the residual stream after
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
        """One dict per layer: paged latent rows, paged keys and values, or
        the convolution tail and the fp32 state of every slot."""
        return [layer.mixer.state_tensors(num_blocks, block_size, num_slots,
                                          device) for layer in self.layers]

    # ----------------------------------------------------------- forward
    def forward(self, input_ids, meta, caches, hidden=None, residual=None):
        # one copy of the stream with weight one: embedding row and its norm
        xs, h = seqmix.hyper_start(input_ids, self.embed_tokens, self.one,
                                   self.layers[0].norm1, self.arch.eps,
                                   self.dtype)
        resid = xs.view(xs.shape[0], xs.shape[2])
        shared: dict = {}
        n = len(self.layers)
        for i, (layer, cache) in enumerate(zip(self.layers, caches)):
            nxt = (self.final_norm if i + 1 == n
                   else self.layers[i + 1].norm1)
            h = layer(resid, h, meta, cache, nxt, shared)
            if self.residual_trace is not None:
                self.residual_trace.append(resid.detach().clone())
        return h

    def compute_logits(self, hidden: torch.Tensor) -> torch.Tensor:
        return self.lm_head(hidden).float()

    # ----------------------------------------------------------- weights
    def load_weights(self, tensors: Iterable[Tuple[str, torch.Tensor]]) -> int:
        """Checkpoint names -> parameters. A mixer's input branches land in
        its layer's merged projection; the layer norms' weights gain the one
        they are stored without; norm weights, step-size biases, decays, skip
        weights and convolution taps are kept in fp32. Second norms of a
        layer without feed-forward are passed over."""
        n = 0
        seen = set()
        # norms around a feed-forward that the layer does not have
        unused = {f"l{i}.norm{q}" for i, layer in enumerate(self.layers)
                  if layer.mlp is None for q in ("2", "2b")}
        for name, t in tensors:
            if name in unused:
                continue
            self._load_one(name, t)
            seen.add(name)
            n += 1
        missing = [k for k in self.expected_tensor_names() if k not in seen]
        if missing:
            raise ValueError(f"checkpoint lacks tensors: {missing[:8]}"
                             f"{' ...' if len(missing) > 8 else ''}")
        for layer in self.layers:
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
            "final.norm": (self.final_norm, ("plus_one",)),
        }
        for i, layer in enumerate(self.layers):
            p = f"l{i}."
            mp = p + "mix."
            mod = layer.mixer
            for q in ("1", "1b", "2", "2b"):
                if layer.mlp is not None or q[0] == "1":
                    out[f"{p}norm{q}"] = (getattr(layer, f"norm{q}"),
                                          ("plus_one",))
            for br in mod.in_names:
                rows = layer.in_proj_rows(br)
                out[mp + br] = (layer.in_proj.weight, rows)
                if br in getattr(mod, "biased", ()):
                    out[mp + br + ".b"] = (layer.in_proj.bias, rows)
            out[mp + "o"] = (mod.o_proj.weight, None)
            if isinstance(mod, LatentAttention):
                out[mp + "dq.norm"] = (mod.q_norm, None)
                out[mp + "uq"] = (mod.uq.weight, None)
                out[mp + "dkv.norm"] = (mod.c_norm, None)
                out[mp + "uk"] = (mod.uk, None)
                out[mp + "uv"] = (mod.uv_t, ("heads_t",))
            elif isinstance(mod, NormedHeadAttention):
                out[mp + "o.b"] = (mod.o_bias, None)
                out[mp + "q.norm"] = (mod.q_norm, None)
                out[mp + "k.norm"] = (mod.k_norm, None)
                if mod.vmix is not None:
                    out[mp + "vmix"] = (mod.vmix, None)
            else:
                out[mp + "conv"] = (mod.conv_w, None)
                out[mp + "conv.b"] = (mod.conv_b, None)
                out[mp + "x"] = (mod.x_proj.weight, None)
                out[mp + "dt"] = (mod.dt_proj.weight, None)
                out[mp + "dt.b"] = (mod.dt_bias, None)
                out[mp + "A_log"] = (mod.a_log, None)
                out[mp + "D"] = (mod.d_skip, None)
            if layer.mlp is not None:
                out[p + "mlp.up"] = (layer.mlp.up_proj.weight, None)
                out[p + "mlp.down"] = (layer.mlp.down_proj.weight, None)
        return out

    @staticmethod
    def _view(param, spec):
        dst = param.data
        if spec is None or spec[0] == "plus_one":
            return dst
        if spec[0] == "heads_t":     # stored [H, in, out] per head
            return dst.transpose(1, 2)
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
        t = t.to(dst.dtype)
        dst.copy_(t + 1.0 if spec == ("plus_one",) else t)

    def export_weights(self) -> Dict[str, torch.Tensor]:
        """Inverse of load_weights (checkpoint naming), for writing
        random-init models to disk."""
        out = {}
        for k, (p, spec) in self._name_map().items():
            t = self._view(p, spec).detach().clone().contiguous()
            if spec is not None and spec[0] == "heads_t":
                t = t.view(-1, t.shape[-1])
            out[k] = t - 1.0 if spec == ("plus_one",) else t
        return out

    def randomize_small_params(self, seed: int = 0) -> None:
        """Random-init use (benchmarks, tests): give norm weights, biases,
        blend factors, step sizes, decays and taps non-trivial values so
        every branch contributes."""
        g = torch.Generator().manual_seed(seed)

        def rnd(p, lo, hi):
            p.data.copy_((torch.rand(p.shape, generator=g) * (hi - lo) + lo)
                         .to(device=p.device, dtype=p.dtype))

        rnd(self.final_norm, 0.8, 1.2)
        for layer in self.layers:
            mod = layer.mixer
            for q in ("1", "1b", "2", "2b"):
                if layer.mlp is not None or q[0] == "1":
                    rnd(getattr(layer, f"norm{q}"), 0.5, 1.5)
            if isinstance(mod, LatentAttention):
                rnd(mod.q_norm, 0.5, 1.5)
                rnd(mod.c_norm, 0.5, 1.5)
            elif isinstance(mod, NormedHeadAttention):
                rnd(layer.in_proj.bias, -0.3, 0.3)
                rnd(mod.o_bias, -0.3, 0.3)
                rnd(mod.q_norm, 0.5, 1.5)
                rnd(mod.k_norm, 0.5, 1.5)
                if mod.vmix is not None:
                    rnd(mod.vmix, 0.2, 0.8)
            else:
                rnd(mod.conv_w, -0.6, 0.6)
                rnd(mod.conv_b, -0.2, 0.2)
                rnd(mod.dt_bias, -4.0, 0.0)
                rnd(mod.a_log, -1.0, 2.0)
                rnd(mod.d_skip, 0.5, 1.5)
