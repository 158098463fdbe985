"""Sufavik through the engine against the float64 oracle in
tests/oracles/sufavik_oracle.py: every mechanism alone, prompts against
token-by-token decoding, portions down to two tokens, unequal batches,
recycled pages and slots, far keys and far memories at page, tile, chunk
and span borders, first tokens, long decoding, odd sizes, both forms of
latent attention, and greedy generation through the scheduler.

The same cases run on the CPU ops (always) and on the HIP kernels (gpu
marker)."""

import json
import math
import os
import subprocess
import sys

import pytest
import torch

from fusioninfer_amd import ops
from fusioninfer_amd.config import CacheConfig, EngineConfig, SchedulerConfig
from fusioninfer_amd.engine.llm_engine import LLMEngine
from fusioninfer_amd.engine.metadata import AttnMetadata
from fusioninfer_amd.engine.sequence import SamplingParams
from fusioninfer_amd.models import registry
from fusioninfer_amd.models.mixers import (
    GatedMemoryConfig,
    GatedMemoryMixer,
    GatedMLP,
    HyperLayer,
    LatentAttention,
    LatentAttentionConfig,
    RoutedExperts,
    SharedExpertMoE,
)
from fusioninfer_amd.ops import seqmix
from tests.oracles import sufavik_oracle as oracle

DEVICES = ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)]
F64 = torch.float64
TOL = 2e-4   # fp32 engine vs float64 oracle, relative
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


# ---------------------------------------------------------------- configs

def rot_cfg(dims, base=300.0, scaling=True, factor=3.0, original=48,
            fast=6.0, slow=1.5):
    r = {"dims": dims, "base": base}
    if scaling:
        r["scaling"] = {"factor": factor, "original": original, "fast": fast,
                        "slow": slow}
    return r


def latent_cfg(heads=3, dim=6, rot_dim=4, vdim=10, kv_rank=14, q_rank=9,
               scale=0.35, rot=None, kv_from=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim,
         "kv_rank": kv_rank, "q_rank": q_rank, "scale": scale,
         "rot": rot or rot_cfg(rot_dim)}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return m


def memory_cfg(heads=2, dim=5, vdim=9, gate_cap=7.0):
    return {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": gate_cap}


def dense_cfg(ff=40):
    return {"kind": "dense", "ff": ff}


def moe_cfg(ff=24, experts=6, identity=3, top=3, shared=20):
    m = {"kind": "moe", "expert": {"ff": ff},
         "router": {"experts": experts, "identity": identity, "top": top}}
    if shared:
        m["shared"] = {"ff": shared}
    return m


def latent(mixer, mlp):
    return {"type": "latent_attention", "mixer": mixer, "mlp": mlp}


def memory(mixer, mlp):
    return {"type": "mlstm", "mixer": mixer, "mlp": mlp}


def small_config():
    """Sizes chosen so that nothing coincides: three copies of the stream,
    every head count and size different, layers that borrow latents (one
    across another owner, with other head sizes), a rotation without
    blend, value sizes above one column tile, a layer without
    feed-forward, routing without identity or shared expert."""
    plain = rot_cfg(6, base=90.0, scaling=False)
    return {
        "architecture": "Sufavik",
        "vocab": 83,
        "width": 44,
        "norm": {"eps": 1e-3},
        "streams": 3,
        "layers": [
            latent(latent_cfg(), dense_cfg()),
            memory(memory_cfg(), moe_cfg()),
            latent(latent_cfg(heads=5, dim=8, vdim=3, q_rank=11, scale=0.2,
                              kv_from=0), None),
            latent(latent_cfg(heads=2, dim=4, rot_dim=6, vdim=7, kv_rank=21,
                              q_rank=16, scale=0.5, rot=plain),
                   moe_cfg(16, 4, 0, 2, 0)),
            memory(memory_cfg(3, 8, 70, 4.0), dense_cfg(24)),
            latent(latent_cfg(heads=4, dim=5, rot_dim=6, vdim=12, kv_rank=21,
                              q_rank=7, scale=0.3, rot=plain, kv_from=3),
                   moe_cfg(12, 3, 1, 1, 28)),
        ],
    }


def make_engine(raw, device, dtype="float32", blocks=64, max_seqs=4,
                seed=0, budget=4096, eager=True):
    mc = registry.model_config_from_dict(raw)
    mc.dtype = dtype
    cfg = EngineConfig(
        model=mc,
        cache=CacheConfig(num_gpu_blocks=blocks, enable_prefix_caching=False),
        scheduler=SchedulerConfig(max_num_seqs=max_seqs,
                                  max_num_batched_tokens=budget,
                                  max_model_len=blocks * 16,
                                  prefill_admission_tokens=0),
        enforce_eager=eager,
        num_state_slots=max_seqs,
        seed=seed,
    )
    eng = LLMEngine(cfg, device=device)
    model = eng.runner.model
    # livelier weights than the 0.02-std init so that every branch matters
    g = torch.Generator().manual_seed(seed + 2)
    for name, p in model.named_parameters():
        if p.dim() >= 2:
            fan = p.shape[-2] if name.endswith("uv_t") else p.shape[-1]
            p.data.copy_((torch.randn(p.shape, generator=g)
                          / math.sqrt(fan)).to(p.dtype).to(p.device))
    model.randomize_small_params(seed + 1)
    for lay in model.layers:
        if isinstance(lay.mlp, SharedExpertMoE):
            lay.mlp.routed.invalidate_packed()
        if isinstance(lay.mixer, LatentAttention):
            lay.mixer.invalidate_packed()
    W = {k: v.detach().cpu().to(F64)
         for k, v in model.export_weights().items()}
    return eng, W


def set_expansion(eng, rows_per_key):
    """Rows per context row from which prompt portions attend in expanded
    form (1: always, a huge value: never)."""
    for lay in eng.runner.model.layers:
        if isinstance(lay.mixer, LatentAttention):
            lay.mixer.expand_rows_per_key = rows_per_key


def row_err(got, want):
    got, want = got.double().cpu(), want.double().cpu()
    d = got - want
    d = d - d.mean(-1, keepdim=True)
    w = want - want.mean(-1, keepdim=True)
    return d.pow(2).mean(-1).sqrt() / w.pow(2).mean(-1).sqrt()


def rel_err(got, want):
    """Mean-free RMS difference relative to the RMS of the expected row."""
    return row_err(got, want).max().item()


def run_schedule(eng, steps):
    """steps: [[(id, tokens, want)], ...] with ('end', id) tuples allowed;
    returns {id: {position: logits}}."""
    got, at = {}, {}
    for step in steps:
        entries = [e for e in step if e[0] != "end"]
        end = [e[1] for e in step if e[0] == "end"]
        out = eng.forced_step(entries, end).cpu()
        row = 0
        for rid, toks, want in entries:
            for w in want:
                got.setdefault(rid, {})[at.get(rid, 0) + w] = out[row]
                row += 1
            at[rid] = at.get(rid, 0) + len(toks)
        for rid in end:
            at.pop(rid, None)
    return got


def tokens(n, seed, vocab=83):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, vocab, (n,), generator=g).tolist()


def mk(v, device):
    return torch.tensor(v, dtype=torch.int32, device=device)


def step_meta(spans, device, bs=16):
    """Metadata of one step, portions first: spans = [(sequence, first
    position, rows)]; sequence s owns pages 64 s .. and state slot s; its
    pages are shuffled."""
    pos, slot_map, row_seq, cu, bts = [], [], [], [0], []
    for i, (s, p0, n) in enumerate(spans):
        g = torch.Generator().manual_seed(s)
        pg = (torch.randperm(64, generator=g) + 64 * s).tolist()
        bts.append(pg)
        for p in range(p0, p0 + n):
            pos.append(p)
            slot_map.append(pg[p // bs] * bs + p % bs)
            row_seq.append(i)
        cu.append(cu[-1] + n)
    meta = AttnMetadata(num_prefill_tokens=len(pos), num_decode_tokens=0,
                        positions=mk(pos, device),
                        slot_mapping=mk(slot_map, device))
    meta.seq_cu = mk(cu, device)
    meta.row_seq = mk(row_seq, device)
    meta.seq_bt = mk(bts, device)
    meta.seq_slots = mk([s for s, _, _ in spans], device)
    meta.max_seq_rows = max(n for _, _, n in spans)
    lead = [(n, p0 + n, bts[i]) for i, (_, p0, n) in enumerate(spans)
            if n > 1]
    assert all(n > 1 for _, _, n in spans[: len(lead)])
    if lead:
        meta.seq_tiles = seqmix.build_attention_tiles(
            [n for n, _, _ in lead], device=device)
        meta.prefill_spans = lead
    return meta


def one_layer(mixer, width, device, seed=0):
    """A mixer behind the merged projection of a layer, with lively
    weights, and its matrices under the oracle's names."""
    layer = HyperLayer(mixer, None, 1, width, 1e-4, torch.float32)
    g = torch.Generator().manual_seed(seed + 5)
    for name, p in layer.named_parameters():
        if p.dim() >= 2:
            fan = p.shape[-2] if name.endswith("uv_t") else p.shape[-1]
            p.data.copy_(torch.randn(p.shape, generator=g) / math.sqrt(fan))
    return layer.to(device), g


def mixer_weights(layer):
    mod = layer.mixer
    W = {}
    for br in mod.in_names:
        a, n = layer.in_proj_rows(br)
        W[br] = layer.in_proj.weight.data[a:a + n]
    W["o"] = mod.o_proj.weight.data
    if isinstance(mod, LatentAttention):
        W.update({"dq.norm": mod.q_norm.data, "uq": mod.uq.weight.data,
                  "uk": mod.uk.data, "uv": mod.uv.data})
        if mod.own_kv:
            W["dkv.norm"] = mod.c_norm.data
    else:
        W.update({"i.b": mod.i_bias.data, "f.b": mod.f_bias.data,
                  "norm": mod.norm_w.data})
    return {k: v.cpu().to(F64) for k, v in W.items()}


def run_mixer(layer, h, steps, device, cache):
    """Feed rows of h {seq: [T, width]} step by step; steps: [[(seq, first
    position, rows)]]."""
    out = {s: torch.zeros(v.shape[0], layer.mixer.o_proj.weight.shape[0])
           for s, v in h.items()}
    for step in steps:
        order = sorted(step, key=lambda e: e[2] == 1)   # portions first
        meta = step_meta(order, device)
        x = torch.cat([h[s][p0:p0 + n] for s, p0, n in order]).to(device)
        parts = layer.in_proj(x).split(layer.sizes, dim=-1)
        y = layer.mixer(parts, meta, cache).cpu()
        a = 0
        for s, p0, n in order:
            out[s][p0:p0 + n] = y[a:a + n]
            a += n
    return out


MIXED_STEPS = [
    [(0, 0, 2), (1, 0, 21)],
    [(0, 2, 1), (1, 21, 2)],
    [(0, 3, 17), (1, 23, 1)],
    [(0, 20, 1), (1, 24, 1)],
    [(0, 21, 19)],
]


# ----------------------------------------------------- mechanisms alone

@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("S", [1, 2, 3, 4, 6, 8])
@pytest.mark.parametrize("T,W", [(5, 24), (3, 101), (4, 1028), (2, 2304),
                                 (1, 4200)])
def test_stream_copies(device, S, T, W):
    g = torch.Generator().manual_seed(S * 7 + W)
    V, eps = 19, 1e-3
    emb = torch.randn(V, W, generator=g)
    ids = torch.randint(0, V, (T,), generator=g)
    vec = lambda n: torch.randn(n, generator=g)
    w1, w2, a1, a2, b = vec(W), vec(W), vec(S), vec(S), vec(S)
    M = torch.randn(S, S, generator=g)
    dev = lambda *ts: [t.to(device) for t in ts]
    ids_d, emb_d, w1_d, w2_d, a1_d, a2_d, b_d, M_d = dev(
        ids, emb, w1, w2, a1, a2, b, M)
    xs, h = seqmix.hyper_start(ids_d, emb_d, a1_d, w1_d, eps, torch.float32)
    want = emb[ids].double()[None].repeat(S, 1, 1)
    assert torch.equal(xs.cpu(), want.transpose(0, 1).float())
    wh = oracle.rms_norm(oracle.read_streams(want, a1.double()), w1.double(),
                         eps)
    assert rel_err(h, wh) < TOL
    # y of one, two and three terms: plain, with a sigmoid gate that is a
    # column of a wider matrix, with a plain coefficient
    ys = [torch.randn(T, W, generator=g) for _ in range(3)]
    gate = torch.randn(T, 5, generator=g)
    coef = torch.randn(T, generator=g)
    gate_d, coef_d = dev(gate, coef)
    ys_d = dev(*ys)
    for n in (1, 2, 3):
        terms = [(ys_d[0], None, False), (ys_d[1], gate_d[:, 3], True),
                 (ys_d[2], coef_d, False)][:n]
        y = ys[0].double()
        if n > 1:
            y = y + torch.sigmoid(gate[:, 3].double())[:, None] * ys[1]
        if n > 2:
            y = y + coef.double()[:, None] * ys[2]
        h = seqmix.hyper_update_(xs, terms, M_d, b_d, a2_d, w2_d, eps,
                                 torch.float32)
        want = oracle.write_streams(want, y, M.double(), b.double())
        got = xs.cpu().transpose(0, 1)
        assert rel_err(got.reshape(S * T, W),
                       want.reshape(S * T, W)) < 1e-5
        wh = oracle.rms_norm(oracle.read_streams(want, a2.double()),
                             w2.double(), eps)
        assert rel_err(h, wh) < TOL
    # bf16 activations: the copies stay fp32, the emitted row is rounded
    xb = xs.clone()
    yb = ys_d[0].to(torch.bfloat16)
    hb = seqmix.hyper_update_(xb, [(yb, None, False)], M_d, b_d, a2_d, w2_d,
                              eps, torch.bfloat16)
    want = oracle.write_streams(xs.cpu().double().transpose(0, 1),
                                yb.cpu().double(), M.double(), b.double())
    assert rel_err(xb.cpu().transpose(0, 1).reshape(S * T, W),
                   want.reshape(S * T, W)) < 1e-5
    wh = oracle.rms_norm(oracle.read_streams(want, a2.double()), w2.double(),
                         eps)
    assert hb.dtype == torch.bfloat16 and rel_err(hb, wh) < 1e-2


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("T,F_", [(3, 10), (5, 64), (2, 1030)])
def test_silu_unit(device, T, F_):
    gu = torch.randn(T, 2 * F_, generator=torch.Generator().manual_seed(F_))
    want = oracle.silu(gu[:, :F_].double()) * gu[:, F_:].double()
    got = seqmix.silu_and_mul((gu * 3).to(device) / 3)
    assert torch.allclose(got.cpu().double(), want, atol=1e-5)


def latent_layer(device, H, dim, rot, vdim, rank, q_rank, own=True,
                 scaling=True, seed=0, width=40, scale=0.27):
    rc = rot_cfg(rot, scaling=scaling)
    sc = rc.get("scaling") or {}
    cfg = LatentAttentionConfig(
        heads=H, dim=dim, rot_dim=rot, vdim=vdim, rank=rank, scale=scale,
        rot_base=rc["base"], sink=False, q_rank=q_rank, head_gate=True,
        rot_factor=sc.get("factor", 1.0),
        rot_original=sc.get("original", 0.0), rot_fast=sc.get("fast", 0.0),
        rot_slow=sc.get("slow", 0.0))
    layer, g = one_layer(
        LatentAttention(cfg, width, 1e-4, torch.float32, own_kv=own), width,
        device, seed)
    mod = layer.mixer
    mod.q_norm.data.copy_(torch.rand(q_rank, generator=g) + 0.5)
    if own:
        mod.c_norm.data.copy_(torch.rand(rank, generator=g) + 0.5)
    m = {"heads": H, "dim": dim, "rot_dim": rot, "vdim": vdim,
         "kv_rank": rank, "scale": scale, "rot": rc}
    return layer, m, g


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("expand", [1, 1 << 30])
@pytest.mark.parametrize("H,dim,rot,vdim,rank,q_rank,scaling", [
    (3, 8, 6, 10, 20, 12, True), (1, 4, 2, 4, 7, 5, False),
    (9, 6, 4, 5, 12, 16, True), (2, 32, 16, 32, 96, 24, True),
    (2, 32, 32, 64, 256, 24, True), (4, 5, 10, 3, 9, 1, True),
    (2, 33, 31 * 2, 1, 1, 7, False), (2, 96, 32, 128, 256, 40, True)])
def test_latent_attention(device, expand, H, dim, rot, vdim, rank, q_rank,
                          scaling):
    """Own latents through mixed steps, then a borrowing layer with other
    head sizes on the same cache; folded form and expanded form."""
    layer, m, g = latent_layer(device, H, dim, rot, vdim, rank, q_rank,
                               scaling=scaling)
    layer.mixer.expand_rows_per_key = expand
    h = {0: torch.randn(40, 40, generator=g),
         1: torch.randn(25, 40, generator=g)}
    cache = layer.mixer.state_tensors(128, 16, 2, device)
    got = run_mixer(layer, h, MIXED_STEPS, device, cache)
    W = mixer_weights(layer)
    held = {}
    for s in h:
        held[s] = oracle.latents(h[s].double(), W, "", m, 1e-4)
        want = oracle.latent_attention_mixer(h[s].double(), W, "", m, 1e-4,
                                             held[s])
        assert rel_err(got[s], want) < TOL, s
    other, m2, g2 = latent_layer(device, H + 2, dim + 1, rot, vdim + 3, rank,
                                 q_rank + 2, own=False, scaling=scaling,
                                 seed=9, scale=0.4)
    other.mixer.expand_rows_per_key = expand
    before = cache["kv"].clone()
    h2 = {s: torch.randn(v.shape, generator=g2) for s, v in h.items()}
    got = run_mixer(other, h2, MIXED_STEPS, device, cache)
    W2 = mixer_weights(other)
    for s in h2:
        want = oracle.latent_attention_mixer(h2[s].double(), W2, "", m2,
                                             1e-4, held[s])
        assert rel_err(got[s], want) < TOL, s
    assert torch.equal(cache["kv"], before)    # a borrower writes nothing


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("expand", [1, 1 << 30])
@pytest.mark.parametrize("hot", [0, 1, 15, 16, 63, 64, 127, 128, 255, 256,
                                 290])
@pytest.mark.parametrize("rows", [1, 2, 43])
def test_far_latent_decides_the_row(device, expand, hot, rows):
    """All queries and one key share a strong direction; the key sits at
    page (16), key-tile (64), row-tile (128) and span (256) borders of a
    shuffled context, and the last rows come as one portion or decoded."""
    H, dim, rot, vdim, rank, q_rank, T = 2, 48, 16, 64, 40, 10, 300
    layer, m, g = latent_layer(device, H, dim, rot, vdim, rank, q_rank,
                               scale=0.15)
    mod = layer.mixer
    mod.expand_rows_per_key = expand
    a, _ = layer.in_proj_rows("dq")
    b, _ = layer.in_proj_rows("dkv")
    w = layer.in_proj.weight.data
    w[a], w[b] = 0, 0
    w[a, 0] = 9.0          # every row's query latent leads with entry 0
    w[b, 1] = 9.0          # the hot row's latent leads with entry 0
    for hh in range(H):
        mod.uq.weight.data[hh * (dim + rot), 0] = 9.0
        mod.uk.data[hh * dim, 0] = 5.0
    mod.invalidate_packed()
    h = torch.randn(T, 40, generator=g)
    h[:, 0] = 2.0
    h[:, 1] *= 0.1
    h[hot, 1] = 3.0
    steps = [[(0, 0, T - rows)], [(0, T - rows, rows)]]
    cache = mod.state_tensors(64, 16, 1, device)
    got = run_mixer(layer, {0: h}, steps, device, cache)[0][T - rows:]
    W = mixer_weights(layer)
    c, kr = oracle.latents(h.double(), W, "", m, 1e-4)
    full = lambda cc, kk: oracle.latent_attention_mixer(
        h[T - rows:].double(), W, "", m, 1e-4, (cc, kk), pos0=T - rows)
    want = full(c, kr)
    assert rel_err(got, want) < TOL
    c2 = c.clone()
    c2[hot] = 0                       # without it the rows are different
    assert row_err(full(c2, kr), want)[-1] > 0.2


def memory_layer(device, H, D, V, cap=6.0, seed=0, width=40, i_bias=0.0,
                 f_bias=2.0):
    layer, g = one_layer(
        GatedMemoryMixer(GatedMemoryConfig(H, D, V, cap), width, 1e-4,
                         torch.float32), width, device, seed)
    mod = layer.mixer
    mod.i_bias.data.copy_(torch.randn(H, generator=g) + i_bias)
    mod.f_bias.data.copy_(torch.randn(H, generator=g) + f_bias)
    mod.norm_w.data.copy_(torch.rand(H * V, generator=g) + 0.5)
    return layer, {"heads": H, "dim": D, "vdim": V, "gate_cap": cap}, g


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("H,D,V,cap,i_bias,f_bias", [
    (2, 6, 9, 6.0, 0.0, 2.0), (1, 1, 1, 2.0, 0.0, 0.0),
    (3, 32, 64, 15.0, -6.0, 3.0), (2, 64, 65, 9.0, 5.0, -3.0),
    (1, 20, 200, 4.0, 0.0, 6.0), (2, 130, 24, 12.0, 1.0, 5.0),
    (1, 300, 12, 12.0, 1.0, 5.0), (5, 16, 33, 30.0, -12.0, -12.0)])
def test_matrix_memory(device, H, D, V, cap, i_bias, f_bias):
    """Portions (chunked on the GPU), two-row portions and decoded rows,
    with leftovers of earlier owners in the slots."""
    layer, m, g = memory_layer(device, H, D, V, cap, i_bias=i_bias,
                               f_bias=f_bias)
    h = {0: torch.randn(40, 40, generator=g) * 2,
         1: torch.randn(25, 40, generator=g) * 2,
         2: torch.randn(215, 40, generator=g) * 2}
    cache = layer.mixer.state_tensors(1, 16, 3, device)
    for v in cache.values():
        v.normal_()
    steps = MIXED_STEPS + [[(2, 0, 131)], [(2, 131, 2)], [(2, 133, 1)],
                           [(2, 134, 1)], [(2, 135, 16)], [(2, 151, 64)]]
    got = run_mixer(layer, h, steps, device, cache)
    W = mixer_weights(layer)
    for s in h:
        want = oracle.memory_mixer(h[s].double(), W, "", m, 1e-4)
        assert rel_err(got[s], want) < TOL, s
    # every workgroup's copy of the normalizer and maximum agrees
    aux = cache["aux"].cpu()
    assert torch.allclose(aux, aux[:, :, :1].expand_as(aux), rtol=1e-5,
                          atol=1e-6)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("hot", [0, 1, 63, 64, 65, 127, 128, 191])
@pytest.mark.parametrize("tail", [1, 2, 70])
def test_far_memory_decides_the_row(device, hot, tail):
    """One token writes with a wide open input gate, all others with a
    hundredth of its weight, and hardly anything is forgotten: its value must show hundreds of
    rows later, wherever it sits in a chunk."""
    H, D, V, T = 2, 16, 40, 330
    layer, m, g = memory_layer(device, H, D, V, cap=12.0)
    a, n = layer.in_proj_rows("i")
    b, _ = layer.in_proj_rows("f")
    w = layer.in_proj.weight.data
    w[a:a + n], w[b:b + n] = 0, 0
    w[a:a + n, 0] = 2.0
    mod = layer.mixer
    mod.i_bias.data.fill_(0.0)
    mod.f_bias.data.fill_(11.0)
    h = torch.randn(T, 40, generator=g)
    h[:, 0] = -1.0
    h[hot, 0] = 1.4
    steps = [[(0, 0, T - tail)]]
    steps += [[(0, T - tail, tail)]] if tail > 1 else [[(0, T - 1, 1)]]
    cache = mod.state_tensors(1, 16, 1, device)
    got = run_mixer(layer, {0: h}, steps, device, cache)[0]
    W = mixer_weights(layer)
    want = oracle.memory_mixer(h.double(), W, "", m, 1e-4)
    assert rel_err(got, want) < TOL
    h2 = h.clone()
    h2[hot, 0] = -1.0
    lost = oracle.memory_mixer(h2.double(), W, "", m, 1e-4)
    assert row_err(lost[-1:], want[-1:]).min() > 0.2


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("E,n_id,k,side", [
    (6, 2, 3, 1), (1, 0, 1, 0), (1, 3, 4, 1), (70, 10, 8, 1), (130, 1, 5, 0),
    (1000, 24, 2, 0), (4, 0, 4, 2)])
def test_corrected_router_with_identity_experts(device, E, n_id, k, side):
    g = torch.Generator().manual_seed(E + n_id)
    T, n = 37, E + n_id
    z = torch.randn(T, n + side, generator=g) * 2
    corr = torch.randn(n, generator=g) * 0.3 - 0.2
    wide = z.to(device)
    w, ids, idw = ops.moe_route_corrected(wide[:, :n], corr.to(device), k, E)
    for t in range(T):
        want = oracle.route(z[t, :n].double(), corr.double(), k)
        assert ids[t].tolist() == [a for a, _ in want]
        assert torch.allclose(w[t].cpu().double(),
                              torch.stack([s for _, s in want]), rtol=1e-4,
                              atol=1e-7)
        wid = sum((float(s) for a, s in want if a >= E), 0.0)
        assert abs(float(idw[t]) - wid) < 1e-5


def _experts_case(device, dtype, width, ff, E, n_id, top, shared, T):
    g = torch.Generator().manual_seed(width + E)
    routed = RoutedExperts(width, ff, E, top, dtype, score="softmax",
                           renorm=False, identity=n_id,
                           side_gates=1 if shared else 0)
    moe = SharedExpertMoE(routed, GatedMLP(width, shared, dtype, act="silu")
                          if shared else None)
    for p in moe.parameters():
        if p.dim() >= 2:
            p.data.copy_((torch.randn(p.shape, generator=g)
                          / math.sqrt(p.shape[-1])).to(p.dtype))
    routed.correction.data.copy_(torch.randn(E + n_id, generator=g) * 0.05)
    W = {"router": routed.router.data[: E + n_id],
         "correction": routed.correction.data}
    for e in range(E):
        W[f"e{e}.gate"] = routed.gate_up.data[e, :ff]
        W[f"e{e}.up"] = routed.gate_up.data[e, ff:]
        W[f"e{e}.down"] = routed.down.data[e]
    mlp = {"router": {"experts": E, "top": top}}
    if shared:
        mlp["shared"] = {"ff": shared}
        s = moe.shared
        W["shared.gate"] = s.gate_up_proj.weight.data[:shared]
        W["shared.up"] = s.gate_up_proj.weight.data[shared:]
        W["shared.down"] = s.down_proj.weight.data
        W["shared.sg"] = routed.router.data[E + n_id:]
    W = {k: v.to(F64) for k, v in W.items()}
    h = torch.randn(T, width, generator=g).to(dtype)
    want = oracle.routed_experts(h.double(), W, "", mlp)
    moe = moe.to(device)
    got = 0
    for rows, coef, sig in moe.terms(h.to(device)):
        v = rows.double()
        if coef is not None:
            c = coef.double()
            v = v * (torch.sigmoid(c) if sig else c)[:, None]
        got = got + v
    return got.cpu(), want


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("width,ff,E,n_id,top,shared", [
    (20, 12, 6, 2, 3, 16), (33, 7, 1, 0, 1, 0), (24, 24, 4, 4, 8, 5),
    (64, 32, 10, 1, 2, 0)])
def test_experts_with_identity_and_shared(device, width, ff, E, n_id, top,
                                          shared):
    got, want = _experts_case(device, torch.float32, width, ff, E, n_id, top,
                              shared, 23)
    assert rel_err(got, want) < TOL


@pytest.mark.gpu
@pytest.mark.parametrize("width,ff,E,n_id,top,shared,T", [
    (128, 64, 8, 2, 2, 64, 40),      # MFMA kernel, 16-row tiles
    (256, 128, 4, 1, 2, 96, 600),    # MFMA kernel, 128-row tiles
    (96, 48, 6, 3, 2, 40, 50)])      # sizes the tiles do not divide
def test_experts_bf16_gpu(width, ff, E, n_id, top, shared, T):
    got, want = _experts_case("cuda", torch.bfloat16, width, ff, E, n_id,
                              top, shared, T)
    assert row_err(got, want).median() < 1e-2
    assert rel_err(got, want) < 4e-2


# ------------------------------------------------------ through the engine

@pytest.fixture(scope="module", params=DEVICES)
def small(request):
    raw = small_config()
    eng, W = make_engine(raw, request.param)
    toks = tokens(70, 11)
    trace = []
    want = oracle.forward(toks, W, raw, trace)
    return raw, eng, W, toks, want, trace


def test_whole_prompt_layers_and_first_tokens(small):
    raw, eng, W, toks, want, layers = small
    model = eng.runner.model
    model.residual_trace = []
    got = run_schedule(eng, [[("a", toks, list(range(len(toks))))],
                             [("end", "a")]])
    trace, model.residual_trace = model.residual_trace, None
    rows = torch.stack([got["a"][p] for p in range(len(toks))])
    assert rel_err(rows, want) < TOL
    assert rel_err(rows[:3], want[:3]) < TOL
    assert len(trace) == len(layers) == len(raw["layers"])
    for got_x, want_x in zip(trace, layers):
        assert rel_err(got_x, want_x) < TOL
    one = run_schedule(eng, [[("b", toks[:1], [0])], [("end", "b")]])
    assert rel_err(one["b"][0][None], want[:1]) < TOL


def test_prefill_against_token_by_token_decoding(small):
    raw, eng, W, toks, want, _ = small
    steps = [[("d", toks[:1], [0])]]
    steps += [[("d", [t], [0])] for t in toks[1:]]
    steps.append([("end", "d")])
    got = run_schedule(eng, steps)
    rows = torch.stack([got["d"][p] for p in range(len(toks))])
    assert rel_err(rows, want) < TOL


@pytest.mark.parametrize("expand", [1, 64, 1 << 30])
@pytest.mark.parametrize("sizes", [[2] * 35, [3, 16, 1, 2, 31, 2, 15],
                                   [33, 2, 35], [64, 2, 2, 2]])
def test_portions_of_several_sizes(small, sizes, expand):
    raw, eng, W, toks, want, _ = small
    assert sum(sizes) == len(toks)
    set_expansion(eng, expand)
    steps, a = [], 0
    for n in sizes:
        steps.append([("p", toks[a:a + n], list(range(n)))])
        a += n
    steps.append([("end", "p")])
    got = run_schedule(eng, steps)
    set_expansion(eng, 64)
    rows = torch.stack([got["p"][p] for p in range(len(toks))])
    assert rel_err(rows, want) < TOL


@pytest.mark.parametrize("expand", [1, 1 << 30])
def test_unequal_batch_equals_each_alone_and_recycles(small, expand):
    raw, eng, W, toks, want, _ = small
    reqs = {"r0": tokens(41, 1), "r1": tokens(5, 2), "r2": tokens(23, 3),
            "r3": tokens(1, 4), "r4": tokens(37, 5), "r5": tokens(18, 6)}
    ref = {k: oracle.forward(v, W, raw) for k, v in reqs.items()}
    all_ = lambda n: list(range(n))
    t = reqs
    steps = [
        [("r0", t["r0"][:7], all_(7)), ("r1", t["r1"][:2], all_(2))],
        [("r0", t["r0"][7:8], [0]), ("r1", t["r1"][2:], all_(3)),
         ("r2", t["r2"][:20], all_(20)), ("r3", t["r3"], [0]),
         ("end", "r1"), ("end", "r3")],
        # r4 and r5 take the slots and pages r1 and r3 gave back
        [("r4", t["r4"][:30], all_(30)), ("r0", t["r0"][8:9], [0]),
         ("r5", t["r5"][:1], [0]), ("r2", t["r2"][20:21], [0])],
        [("r5", t["r5"][1:2], [0]), ("r0", t["r0"][9:41], all_(32)),
         ("r2", t["r2"][21:], all_(2)), ("r4", t["r4"][30:31], [0]),
         ("end", "r0"), ("end", "r2")],
        [("r4", t["r4"][31:], all_(6)), ("r5", t["r5"][2:], all_(16)),
         ("end", "r4"), ("end", "r5")],
    ]
    set_expansion(eng, expand)
    free_before = (eng.block_manager.num_free(), eng.state_manager.num_free())
    got = run_schedule(eng, steps)
    set_expansion(eng, 64)
    for k, v in reqs.items():
        rows = torch.stack([got[k][p] for p in range(len(v))])
        assert rel_err(rows, ref[k]) < TOL, k
    assert (eng.block_manager.num_free(),
            eng.state_manager.num_free()) == free_before


def test_slot_and_pages_reused_by_a_shorter_request(small):
    """A long request leaves its memory and pages behind; the next one in
    the same slot and pages must start from nothing, and one that is left
    out of a step must find its own again."""
    raw, eng, W, toks, want, _ = small
    run_schedule(eng, [[("x", tokens(60, 9), [])], [("end", "x")]])
    got = run_schedule(eng, [[("y", toks[:2], [0, 1])],
                             [("z", tokens(5, 8), [])],
                             [("y", toks[2:9], list(range(7)))],
                             [("end", "y"), ("end", "z")]])
    rows = torch.stack([got["y"][p] for p in range(9)])
    assert rel_err(rows, want[:9]) < TOL


def test_greedy_generation_through_scheduler(small):
    raw, eng, W, toks, want, _ = small
    prompts = [toks[:13], toks[20:23], toks[30:51]]
    n_new = 12
    outs = eng.generate(prompts, SamplingParams(max_tokens=n_new))
    for p, o in zip(prompts, outs):
        assert o.output_token_ids == oracle.greedy(p, W, raw, n_new)
    assert eng.state_manager.num_free() == eng.state_manager.num_slots


def test_generation_with_small_token_budget_chunks_prompts():
    """The scheduler's own chunked prefill (budget 8 tokens a step) and
    more requests than slots."""
    raw = small_config()
    eng, W = make_engine(raw, "cpu", max_seqs=2, budget=8, seed=3)
    prompts = [tokens(21, 31), tokens(9, 32), tokens(14, 33)]
    outs = eng.generate(prompts, SamplingParams(max_tokens=6))
    for p, o in zip(prompts, outs):
        assert o.output_token_ids == oracle.greedy(p, W, raw, 6)


@pytest.mark.parametrize("device", DEVICES)
def test_long_decoding_past_pages_and_spans(device):
    raw = {
        "architecture": "Sufavik", "vocab": 50, "width": 32,
        "norm": {"eps": 1e-5}, "streams": 2,
        "layers": [
            latent(latent_cfg(heads=2, dim=8, rot_dim=8, vdim=16, kv_rank=24,
                              q_rank=12, scale=0.3),
                   moe_cfg(16, 4, 1, 2, 12)),
            memory(memory_cfg(2, 16, 16, 10.0), dense_cfg(16)),
            latent(latent_cfg(heads=3, dim=8, rot_dim=8, vdim=8, kv_rank=24,
                              q_rank=10, scale=0.25, kv_from=0), None),
        ],
    }
    eng, W = make_engine(raw, device, blocks=24)
    toks = tokens(300, 21, vocab=50)
    want = oracle.forward(toks, W, raw)
    steps = [[("a", toks[:10], list(range(10)))]]
    steps += [[("a", [t], [0])] for t in toks[10:]]
    got = run_schedule(eng, steps)
    rows = torch.stack([got["a"][p] for p in range(len(toks))])
    assert rel_err(rows, want) < TOL


@pytest.mark.parametrize("device", DEVICES)
def test_values_that_could_hide_faults(device):
    """One copy of the stream, eight copies, single heads, ranks of one,
    one expert, only identity experts next to it, all outputs chosen, no
    identity, no shared expert, no feed-forward at all, no frequency
    blend, a blend that touches no pair, memories only."""
    toks = tokens(24, 7, vocab=31)
    base = {"architecture": "Sufavik", "vocab": 31, "width": 16,
            "norm": {"eps": 1e-6}}
    variants = [
        dict(streams=1, layers=[latent(latent_cfg(1, 4, 2, 4, 1, 1, 1.0),
                                       dense_cfg(8))]),
        dict(streams=8, layers=[
            memory(memory_cfg(1, 1, 1, 1.0), moe_cfg(8, 1, 3, 1, 4)),
            memory(memory_cfg(4, 4, 4, 20.0), None)]),
        dict(streams=2, layers=[
            latent(latent_cfg(2, 4, 4, 4, 8, 8, 0.5,
                              rot_cfg(4, scaling=False)),
                   moe_cfg(8, 3, 2, 5, 0)),
            latent(latent_cfg(1, 6, 4, 2, 8, 3, 0.9,
                              rot_cfg(4, scaling=False), kv_from=0),
                   moe_cfg(4, 4, 0, 4, 8))]),
        dict(streams=5, layers=[
            memory(memory_cfg(2, 3, 5, 3.0), None),
            latent(latent_cfg(2, 4, 4, 4, 8, 8, 0.5,
                              rot_cfg(4, factor=1.0)), None)]),
        dict(streams=4, layers=[
            latent(latent_cfg(2, 4, 8, 4, 8, 8, 0.5,
                              rot_cfg(8, original=4096, fast=1e6,
                                      slow=1e5)), moe_cfg(8, 2, 1, 1, 8))]),
    ]
    for i, extra in enumerate(variants):
        raw = dict(base, **extra)
        eng, W = make_engine(raw, device, blocks=8, seed=i)
        want = oracle.forward(toks, W, raw)
        got = run_schedule(eng, [[("a", toks[:2], [0, 1])],
                                 [("a", toks[2:19], list(range(17)))],
                                 [("a", toks[19:20], [0])],
                                 [("a", toks[20:], list(range(4)))]])
        rows = torch.stack([got["a"][p] for p in range(len(toks))])
        assert rel_err(rows, want) < TOL, i


def test_config_is_checked():
    def refused(change):
        raw = small_config()
        change(raw)
        with pytest.raises(ValueError):
            make_engine(raw, "cpu")

    def set_(path, value):
        def change(raw):
            x = raw
            for k in path[:-1]:
                x = x[k]
            x[path[-1]] = value
        return change

    refused(set_(["layers", 2, "mixer", "kv_from"], 2))
    refused(set_(["layers", 2, "mixer", "kv_from"], 1))   # not a latent layer
    refused(set_(["layers", 5, "mixer", "kv_from"], 2))   # a borrower itself
    refused(set_(["layers", 2, "mixer", "kv_rank"], 15))
    refused(set_(["layers", 2, "mixer", "rot", "base"], 77.0))
    refused(set_(["layers", 1, "mlp", "router", "top"], 10))
    refused(set_(["layers", 1, "type"], "convolution"))
    refused(set_(["layers", 0, "mlp", "kind"], "sparse"))
    refused(set_(["streams"], 0))


def test_cache_and_state_declarations():
    raw = small_config()
    eng, _ = make_engine(raw, "cpu", blocks=8)
    caches = eng.runner.kv_caches
    assert caches[2] is caches[0] and caches[5] is caches[3]
    assert caches[0]["kv"].shape == (8, 1, 16, 18)
    assert caches[3]["kv"].shape == (8, 1, 16, 27)
    assert caches[4]["mem"].shape == (4, 3, 8, 70)
    assert caches[4]["mem"].dtype == torch.float32
    assert eng.runner.model.kv_block_bytes(16) == 16 * (18 + 27) * 4


def _write_checkpoint(tmp_path, raw, W):
    from safetensors.torch import save_file

    d = tmp_path / "model"
    d.mkdir()
    (d / "config.json").write_text(json.dumps(raw))
    save_file({k: v.to(torch.bfloat16).contiguous() for k, v in W.items()},
              str(d / "model.safetensors"))
    return str(d)


def test_checkpoint_directory_roundtrip(tmp_path):
    raw = small_config()
    eng, W = make_engine(raw, "cpu", seed=5)
    path = _write_checkpoint(tmp_path, raw, W)
    mc = registry.get_model_config(path)
    assert mc.architecture == "Sufavik" and mc.model_path == path
    assert registry.required_extensions(mc) == ("seqmix", "moe")
    mc.dtype = "float32"
    cfg = EngineConfig(
        model=mc, cache=CacheConfig(num_gpu_blocks=16,
                                    enable_prefix_caching=False),
        scheduler=SchedulerConfig(max_num_seqs=2, max_num_batched_tokens=256,
                                  max_model_len=256), enforce_eager=True,
        num_state_slots=2)
    eng2 = LLMEngine(cfg, device="cpu")
    Wb = {k: v.to(torch.bfloat16).to(F64) for k, v in W.items()}
    toks = tokens(20, 3)
    got = run_schedule(eng2, [[("a", toks, list(range(20)))]])
    rows = torch.stack([got["a"][p] for p in range(20)])
    assert rel_err(rows, oracle.forward(toks, Wb, raw)) < TOL
    # a checkpoint that lacks a tensor, or holds an unknown one, is refused
    from safetensors.torch import load_file, save_file

    t = load_file(os.path.join(path, "model.safetensors"))
    held = t.pop("l1.hc2.mix")
    save_file(t, os.path.join(path, "model.safetensors"))
    with pytest.raises(ValueError):
        LLMEngine(cfg, device="cpu")
    t["l1.hc2.mix"] = held
    t["l2.mix.dkv"] = t["l0.mix.dkv"].clone()   # a borrower has none
    save_file(t, os.path.join(path, "model.safetensors"))
    with pytest.raises(ValueError):
        LLMEngine(cfg, device="cpu")


def test_schedule_replay_program(tmp_path):
    """bin/trace_run as a subprocess on a checkpoint directory, with a
    cache pool smaller than the sum of its requests."""
    raw = small_config()
    eng, W = make_engine(raw, "cpu", seed=6)
    path = _write_checkpoint(tmp_path, raw, W)
    Wb = {k: v.to(torch.bfloat16).to(F64) for k, v in W.items()}
    a, b, c = tokens(50, 1), tokens(33, 2), tokens(40, 3)
    steps = [
        {"step": 0, "entries": [{"id": "a", "tokens": a[:30], "want": [29]},
                                {"id": "b", "tokens": b[:2], "want": [0, 1]}],
         "end": []},
        {"step": 1, "entries": [{"id": "a", "tokens": a[30:31], "want": [0]},
                                {"id": "b", "tokens": b[2:], "want": [30]}],
         "end": ["b"]},
        {"step": 2, "entries": [{"id": "a", "tokens": a[31:], "want": []}],
         "end": ["a"]},
        {"step": 3, "entries": [{"id": "c", "tokens": c, "want": [0, 39]}],
         "end": ["c"]},
    ]
    out = tmp_path / "out"
    p = subprocess.run(
        [sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model",
         path, "--dtype", "float32", "--out", str(out), "--max-tokens", "96",
         "--device", "cpu"],
        input="\n".join(json.dumps(s) for s in steps) + "\n",
        capture_output=True, text=True, timeout=300)
    assert p.returncode == 0, p.stderr[-2000:]
    assert [l for l in p.stdout.split("\n") if l.startswith("done")] == [
        "done 0", "done 1", "done 2", "done 3"]
    import numpy as np

    V = raw["vocab"]
    wa, wb, wc = (oracle.forward(t, Wb, raw) for t in (a, b, c))
    g0 = torch.from_numpy(np.fromfile(out / "0.f32", "<f4").reshape(-1, V))
    g1 = torch.from_numpy(np.fromfile(out / "1.f32", "<f4").reshape(-1, V))
    g3 = torch.from_numpy(np.fromfile(out / "3.f32", "<f4").reshape(-1, V))
    assert not (out / "2.f32").exists()
    assert rel_err(g0, torch.stack([wa[29], wb[0], wb[1]])) < TOL
    assert rel_err(g1, torch.stack([wa[30], wb[32]])) < TOL
    assert rel_err(g3, torch.stack([wc[0], wc[39]])) < TOL


def test_bf16_mode_stays_close_to_oracle():
    raw = small_config()
    eng, W = make_engine(raw, "cpu", dtype="bfloat16", seed=2)
    toks = tokens(40, 5)
    want = oracle.forward(toks, W, raw)
    got = run_schedule(eng, [[("a", toks[:17], list(range(17)))],
                             [("a", toks[17:], list(range(23)))]])
    rows = torch.stack([got["a"][p] for p in range(40)])
    assert row_err(rows, want).median() < 0.05


# ------------------------------------------------------------- GPU only

def tiled_config():
    """Sizes with MFMA tile kernels in both forms of latent attention and
    chunk kernels of the memory, expert sizes the MFMA grouped GEMM takes."""
    r = rot_cfg(32, base=10000.0, factor=2.0, original=128, fast=16.0,
                slow=1.0)
    big = dict(dim=32, rot_dim=32, vdim=64, kv_rank=256, q_rank=48,
               scale=0.125, rot=r)
    return {
        "architecture": "Sufavik", "vocab": 300, "width": 128,
        "norm": {"eps": 1e-5}, "streams": 2,
        "layers": [
            latent(latent_cfg(heads=4, **big), dense_cfg(192)),
            memory(memory_cfg(2, 64, 128, 15.0), moe_cfg(64, 8, 2, 2, 64)),
            latent(latent_cfg(heads=2, kv_from=0, **dict(
                big, dim=96, vdim=128)), moe_cfg(64, 4, 1, 1, 96)),
        ],
    }


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("expand", [1, 64, 1 << 30])
def test_gpu_engine_matches_oracle_at_tiled_sizes(dtype, expand):
    raw = tiled_config()
    eng, W = make_engine(raw, "cuda", dtype=dtype, blocks=80)
    set_expansion(eng, expand)
    a, b = tokens(520, 1, 300), tokens(150, 2, 300)
    wa, wb = oracle.forward(a, W, raw), oracle.forward(b, W, raw)
    ask = lambda n, k=16: list(range(0, n, max(n // k, 1)))
    steps = [
        [("a", a[:300], ask(300)), ("b", b[:2], [0, 1])],
        [("a", a[300:430], ask(130)), ("b", b[2:3], [0])],
        [("b", b[3:140], ask(137)), ("a", a[430:431], [0])],
    ]
    steps += [[("a", [x], [0]), ("b", [y], [0])]
              for x, y in zip(a[431:441], b[140:150])]
    steps.append([("a", a[441:], ask(79)), ("end", "a"), ("end", "b")])
    got = run_schedule(eng, steps)
    for rid, want in (("a", wa), ("b", wb)):
        ps = sorted(got[rid])
        err = row_err(torch.stack([got[rid][p] for p in ps]), want[ps])
        if dtype == "float32":
            assert err.max() < TOL, rid
        else:
            assert err.median() < 0.05, rid


@pytest.mark.gpu
def test_hipgraph_decode_replays_match_oracle():
    raw = small_config()
    eng, W = make_engine(raw, "cuda", eager=False, blocks=32)
    reqs = [tokens(19, 1), tokens(33, 2), tokens(9, 3)]
    want = [oracle.forward(t, W, raw) for t in reqs]
    steps = [[(f"r{i}", t[:-8], []) for i, t in enumerate(reqs)]]
    for k in range(8, 0, -1):
        steps.append([(f"r{i}", [t[len(t) - k]], [0])
                      for i, t in enumerate(reqs)])
    got = run_schedule(eng, steps)
    for i, t in enumerate(reqs):
        ps = sorted(got[f"r{i}"])
        assert ps == list(range(len(t) - 8, len(t)))
        rows = torch.stack([got[f"r{i}"][p] for p in ps])
        assert rel_err(rows, want[i][ps]) < TOL


@pytest.mark.gpu
def test_generation_with_graph_replay():
    raw = small_config()
    eng, W = make_engine(raw, "cuda", eager=False, max_seqs=2, budget=16,
                         seed=4)
    prompts = [tokens(21, 31), tokens(9, 32), tokens(14, 33)]
    outs = eng.generate(prompts, SamplingParams(max_tokens=10))
    for p, o in zip(prompts, outs):
        assert o.output_token_ids == oracle.greedy(p, W, raw, 10)
