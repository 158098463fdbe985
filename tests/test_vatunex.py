"""Vatunex through the engine against the float64 oracle in
tests/oracles/vatunex_oracle.py: every mechanism alone, prompts against
token-by-token decoding, portions down to two tokens, unequal batches,
recycled pages and slots, far keys and far memories at page, window, tile,
segment and span borders, first tokens, long decoding, odd sizes, both
forms of latent attention, and greedy generation through the scheduler.

The same cases run on the CPU ops (always) and on the HIP kernels (gpu
marker)."""

import json
import math
import os
import subprocess
import sys

import pytest
import torch

from fusioninfer_amd.config import CacheConfig, EngineConfig, SchedulerConfig
from fusioninfer_amd.engine.llm_engine import LLMEngine
from fusioninfer_amd.engine.metadata import AttnMetadata
from fusioninfer_amd.engine.sequence import SamplingParams
from fusioninfer_amd.models import registry
from fusioninfer_amd.models.mixers import (
    LatentAttention,
    LatentAttentionConfig,
    NormedHeadAttention,
    NormedHeadAttentionConfig,
    SandwichNormLayer,
    SelectiveScanConfig,
    SelectiveScanMixer,
)
from fusioninfer_amd.ops import seqmix
from tests.oracles import vatunex_oracle as oracle

DEVICES = ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)]
F64 = torch.float64
TOL = 2e-4   # fp32 engine vs float64 oracle, relative
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


# ---------------------------------------------------------------- configs

def latent_cfg(heads=3, dim=6, rot_dim=4, vdim=10, kv_rank=14, q_rank=9,
               scale=0.35, base=300.0, window=7):
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim,
         "kv_rank": kv_rank, "q_rank": q_rank, "scale": scale,
         "rot": {"base": base, "dims": rot_dim}}
    if window:
        m["mask"] = {"size": window}
    return m


def attention_cfg(heads=6, kv_heads=2, dim=10, vdim=7, rot_dims=6,
                  base=150.0, scale=0.3, v_mix=True, scaling=(3.0, 1.5, 5.0,
                                                              40.0)):
    rot = {"base": base, "dims": rot_dims}
    if scaling:
        factor, low, high, original = scaling
        rot["scaling"] = {"factor": factor, "low": low, "high": high,
                          "original": original}
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
            "rot": rot, "scale": scale, "v_mix": v_mix}


def scan_cfg(inner=36, state=5, dt_rank=3, conv=3):
    return {"inner": inner, "state": state, "dt_rank": dt_rank, "conv": conv}


def lay(kind, mixer, ff=40):
    return {"type": kind, "mixer": mixer,
            "mlp": {"kind": "dense", "ff": ff} if ff else None}


latent = lambda m, ff=40: lay("latent_attention", m, ff)
attn = lambda m, ff=40: lay("attention", m, ff)
scan = lambda m, ff=40: lay("mamba1", m, ff)


def small_config():
    """Sizes chosen so that nothing coincides: other head counts, sizes and
    windows in every layer, a layer without feed-forward, an attention
    layer without blending between those with, two recurrences of other
    sizes and taps."""
    return {
        "architecture": "Vatunex",
        "vocab": 83,
        "width": 44,
        "norm": {"eps": 1e-3},
        "layers": [
            scan(scan_cfg(), 24),
            latent(latent_cfg()),
            attn(attention_cfg(), 52),
            latent(latent_cfg(heads=2, dim=5, rot_dim=6, vdim=3, kv_rank=21,
                              q_rank=16, scale=0.5, base=90.0, window=19),
                   None),
            attn(attention_cfg(4, 4, 5, 6, 4, 70.0, 0.6, v_mix=False,
                               scaling=None), 20),
            scan(scan_cfg(50, 9, 7, 5), None),
            attn(attention_cfg(7, 1, 9, 14, 8, 400.0, 0.25), 16),
        ],
    }


def randomize(model, seed):
    """Livelier weights than the 0.02-std init so that every branch
    matters."""
    g = torch.Generator().manual_seed(seed + 2)
    for name, p in model.named_parameters():
        if p.dim() >= 2:
            fan = p.shape[-2] if name.endswith("uv_t") else p.shape[-1]
            p.data.copy_((torch.randn(p.shape, generator=g)
                          / math.sqrt(fan)).to(p.dtype).to(p.device))
    model.randomize_small_params(seed + 1)
    for layer in model.layers:
        if isinstance(layer.mixer, LatentAttention):
            layer.mixer.invalidate_packed()


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
    randomize(model, seed)
    W = {k: v.detach().cpu().to(F64)
         for k, v in model.export_weights().items()}
    return eng, W


def set_expansion(eng, rows_per_key):
    """Rows per context row from which prompt portions attend in expanded
    form (1: soon, a huge value: never)."""
    for layer in eng.runner.model.layers:
        if isinstance(layer.mixer, LatentAttention):
            layer.mixer.expand_rows_per_key = rows_per_key


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


def stacked(got, n):
    return torch.stack([got[p] for p in range(n)])


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
    weights."""
    layer = SandwichNormLayer(mixer, None, width, 1e-4, torch.float32)
    g = torch.Generator().manual_seed(seed + 5)
    for name, p in layer.named_parameters():
        if p.dim() >= 2:
            fan = p.shape[-2] if name.endswith("uv_t") else p.shape[-1]
            p.data.copy_(torch.randn(p.shape, generator=g) / math.sqrt(fan))
    return layer.to(device), g


def mixer_weights(layer):
    """A layer's matrices under the oracle's names."""
    mod = layer.mixer
    W = {"o": mod.o_proj.weight.data}
    for br in mod.in_names:
        a, n = layer.in_proj_rows(br)
        W[br] = layer.in_proj.weight.data[a:a + n]
        if br in getattr(mod, "biased", ()):
            W[br + ".b"] = layer.in_proj.bias.data[a:a + n]
    if isinstance(mod, LatentAttention):
        W.update({"dq.norm": mod.q_norm.data, "uq": mod.uq.weight.data,
                  "uk": mod.uk.data, "uv": mod.uv.data,
                  "dkv.norm": mod.c_norm.data})
    elif isinstance(mod, NormedHeadAttention):
        W.update({"o.b": mod.o_bias.data, "q.norm": mod.q_norm.data,
                  "k.norm": mod.k_norm.data})
        if mod.vmix is not None:
            W["vmix"] = mod.vmix.data
    else:
        W.update({"conv": mod.conv_w.data, "conv.b": mod.conv_b.data,
                  "x": mod.x_proj.weight.data, "dt": mod.dt_proj.weight.data,
                  "dt.b": mod.dt_bias.data, "A_log": mod.a_log.data,
                  "D": mod.d_skip.data})
    return {k: v.cpu().to(F64) for k, v in W.items()}


def run_mixer(layer, h, steps, device, cache, shared=None):
    """Feed rows of h {seq: [T, width]} step by step; steps: [[(seq, first
    position, rows)]]. ``shared``: {seq: [T, *] first values} or None."""
    out = {s: torch.zeros(v.shape[0], layer.mixer.o_proj.weight.shape[0])
           for s, v in h.items()}
    for step in steps:
        order = sorted(step, key=lambda e: e[2] == 1)   # portions first
        meta = step_meta(order, device)
        x = torch.cat([h[s][p0:p0 + n] for s, p0, n in order]).to(device)
        parts = layer.in_proj(x).split(layer.sizes, dim=-1)
        if isinstance(layer.mixer, NormedHeadAttention):
            hand = {}
            if shared is not None:
                hand["v_first"] = torch.cat(
                    [shared[s][p0:p0 + n] for s, p0, n in order]).to(device)
            y = layer.mixer(parts, meta, cache, hand).cpu()
        else:
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
@pytest.mark.parametrize("T,W", [(5, 24), (3, 101), (4, 1028), (2, 2304),
                                 (2, 4100), (1, 9000), (1, 8192)])
def test_norms_on_both_sides(device, T, W):
    g = torch.Generator().manual_seed(W)
    eps = 0.05
    x = torch.randn(T, W, generator=g)
    y = torch.randn(T, W, generator=g) * 0.3
    w1, w2 = torch.randn(W, generator=g), torch.randn(W, generator=g)
    for dt in (torch.float32, torch.bfloat16):
        r = x.to(device).clone()
        yd = y.to(dt).to(device)
        h = seqmix.norm_residual_norm_(r, yd, w1.to(device), w2.to(device),
                                       eps, dt)
        want = x.double() + oracle.rms_norm(yd.cpu().double(), w1.double(),
                                            eps)
        assert rel_err(r, want) < 1e-5       # the stream stays fp32
        wh = oracle.rms_norm(want, w2.double(), eps)
        assert h.dtype == dt
        assert rel_err(h, wh) < (1e-5 if dt == torch.float32 else 1e-2)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("T,N", [(3, 10), (5, 64), (1, 1), (2, 1030)])
def test_gelu(device, T, N):
    x = torch.randn(T, N, generator=torch.Generator().manual_seed(N)) * 3
    x[0, 0] = -40.0
    got = seqmix.gelu_tanh(x.to(device)).cpu()
    assert torch.allclose(got.double(), oracle.gelu_tanh(x.double()),
                          atol=1e-6, rtol=1e-5)


@pytest.mark.parametrize("dims,base,factor,low,high,original", [
    (24, 500.0, 4.0, 1.0, 4.0, 64.0), (8, 1e4, 8.0, 1.0, 1.0, 300.0),
    (64, 5e5, 32.0, 0.5, 9.0, 8192.0), (6, 30.0, 2.0, 1e-4, 2e-4, 10.0),
    (6, 30.0, 2.0, 1e4, 2e4, 10.0), (2, 7.0, 3.0, 1.0, 4.0, 12.0),
    (10, 100.0, 1.0, 1.0, 4.0, 50.0), (12, 100.0, 1.0, 1.0, 1.0, 0.0)])
def test_stretched_frequencies(dims, base, factor, low, high, original):
    rot = {"dims": dims, "base": base}
    if original:
        rot["scaling"] = {"factor": factor, "low": low, "high": high,
                          "original": original}
    want = torch.tensor(oracle.rotary_frequencies(rot), dtype=F64)
    got = seqmix.stretched_rotary(dims, base, factor, low, high, original)
    assert torch.allclose(got.double(), want, rtol=1e-6)


def test_stretched_frequencies_keep_blend_and_divide():
    """One model of frequencies in which all three cases occur."""
    plain = seqmix.stretched_rotary(32, 1000.0)
    got = seqmix.stretched_rotary(32, 1000.0, 8.0, 1.0, 6.0, 200.0)
    turns = 200.0 * plain.double() / (2 * math.pi)
    assert (turns > 6).any() and (turns < 1).any()
    mid = (turns < 6) & (turns > 1)
    assert mid.sum() >= 2
    assert torch.equal(got[turns > 6], plain[turns > 6])
    assert torch.allclose(got[turns < 1] * 8, plain[turns < 1])
    assert (got[mid] < plain[mid]).all() and (got[mid] > plain[mid] / 8).all()


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("H,G,D,n,V,T", [
    (4, 2, 12, 4, 8, 9), (3, 1, 7, 2, 5, 6), (5, 5, 64, 32, 64, 4),
    (2, 1, 80, 20, 48, 1027), (1, 1, 2, 1, 1, 3), (6, 2, 10, 0, 12, 5),
    (2, 2, 520, 260, 4, 3), (1, 1, 301, 77, 9, 3), (3, 1, 40, 4, 3, 1026)])
def test_head_norms_rotation_and_blended_values(device, H, G, D, n, V, T):
    """Column slices of one wide row, a padding row, positions that do not
    start at 0, with and without values to blend in."""
    g = torch.Generator().manual_seed(D + H)
    eps, bs = 1e-3, 16
    wide = torch.randn(T, H * D + G * (D + V) + 3, generator=g)
    first = torch.randn(T, G * V + 5, generator=g)
    q_w, k_w = torch.rand(D, generator=g) + .5, torch.rand(D, generator=g) + .5
    lam = torch.tensor(0.37)
    freqs = [0.9 ** i for i in range(n)]
    pos = torch.arange(T) + 11
    slots = torch.randperm(2 * ((T + 15) // 16) * 16, generator=g)[:T].int()
    slots[T // 2] = -1
    blocks = 2 * ((T + 15) // 16)
    wd = wide.to(device)
    q, k, v = (wd[:, :H * D], wd[:, H * D:(H + G) * D],
               wd[:, (H + G) * D:(H + G) * D + G * V])
    for blend in (False, True):
        kc = torch.full((blocks, G, bs, D), 7.0, device=device)
        vc = torch.full((blocks, G, bs, V), 7.0, device=device)
        got = seqmix.headnorm_rope_cache_(
            q, k, v, first.to(device)[:, 2:2 + G * V] if blend else None,
            lam.to(device), pos.int().to(device), q_w.to(device),
            k_w.to(device), eps, torch.tensor(freqs).to(device), kc, vc,
            slots.to(device), H, G, D, V).cpu()
        for t in sorted({0, 1, 2, T // 2, T - 2, T - 1}):
            row = wide[t].double()

            def turned(x, w):
                return oracle.rotate_half(
                    oracle.rms_norm(x, w.double(), eps), float(pos[t]),
                    [float(torch.tensor(f)) for f in freqs])

            for h in range(H):
                want = turned(row[h * D:(h + 1) * D], q_w)
                assert torch.allclose(got[t, h].double(), want, atol=2e-4)
            s = int(slots[t])
            if s < 0:
                continue
            for a in range(G):
                o = H * D + a * D
                want = turned(row[o:o + D], k_w)
                assert torch.allclose(kc[s // bs, a, s % bs].cpu().double(),
                                      want, atol=2e-4)
                o = (H + G) * D + a * V
                want = row[o:o + V]
                if blend:
                    want = oracle.mix_values(
                        want, first[t, 2 + a * V:2 + (a + 1) * V].double(),
                        lam.double())
                assert torch.allclose(vc[s // bs, a, s % bs].cpu().double(),
                                      want, atol=1e-5)
        # nothing but the rows' own slots was written
        used = set(slots.tolist()) - {-1}
        free = [s for s in range(blocks * bs) if s not in used][:20]
        for s in free:
            assert (kc[s // bs, :, s % bs] == 7).all()
            assert (vc[s // bs, :, s % bs] == 7).all()


def latent_layer(device, H, dim, rot, vdim, rank, q_rank, window, seed=0,
                 width=40, scale=0.27):
    layer, g = one_layer(LatentAttention(LatentAttentionConfig(
        heads=H, dim=dim, rot_dim=rot, vdim=vdim, rank=rank, scale=scale,
        rot_base=250.0, sink=False, q_rank=q_rank, rot_half=True,
        window=window), width, 1e-4, torch.float32), width, device, seed)
    mod = layer.mixer
    mod.q_norm.data.copy_(torch.rand(q_rank, generator=g) + 0.5)
    mod.c_norm.data.copy_(torch.rand(rank, generator=g) + 0.5)
    return layer, latent_cfg(H, dim, rot, vdim, rank, q_rank, scale, 250.0,
                             window), g


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("expand", [0, 1 << 30])
@pytest.mark.parametrize("H,dim,rot,vdim,rank,q_rank,window", [
    (3, 8, 6, 10, 20, 12, 7), (1, 4, 2, 4, 7, 5, 1), (9, 6, 4, 5, 12, 16, 0),
    (2, 32, 32, 64, 112, 24, 17), (2, 32, 32, 64, 256, 24, 33),
    (4, 5, 10, 3, 9, 1, 2), (2, 33, 62, 1, 1, 7, 16),
    (2, 96, 32, 128, 256, 40, 10)])
def test_windowed_latent_attention(device, expand, H, dim, rot, vdim, rank,
                                   q_rank, window):
    layer, m, g = latent_layer(device, H, dim, rot, vdim, rank, q_rank,
                               window)
    layer.mixer.expand_rows_per_key = expand
    h = {0: torch.randn(40, 40, generator=g),
         1: torch.randn(25, 40, generator=g)}
    cache = layer.mixer.state_tensors(128, 16, 2, device)
    got = run_mixer(layer, h, MIXED_STEPS, device, cache)
    W = mixer_weights(layer)
    for s in h:
        want = oracle.latent_attention_mixer(h[s].double(), W, "", m, 1e-4)
        assert rel_err(got[s], want) < TOL, s


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("expand", [0, 1 << 30])
@pytest.mark.parametrize("rows", [1, 2, 43])
@pytest.mark.parametrize("window,back", [
    (1, 0), (2, 1), (16, 15), (17, 16), (45, 44), (64, 63), (65, 64),
    (130, 129), (257, 256), (280, 200), (0, 299)])
def test_strong_latent_at_the_window_edge(device, expand, rows, window,
                                          back):
    """One key outweighs all others. It sits ``back`` before the last row,
    the farthest place that row's window reaches (or far inside it), and is
    invisible from one place farther. The last rows come as one portion or
    decoded."""
    H, dim, rot, vdim, rank, q_rank, T = 2, 48, 16, 64, 40, 10, 300
    layer, m, g = latent_layer(device, H, dim, rot, vdim, rank, q_rank,
                               window, scale=0.15)
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
    base = torch.randn(T, 40, generator=g)
    base[:, 0] = 2.0
    base[:, 1] *= 0.1
    cases = [T - 1 - back]
    if window and back == window - 1 and T - 2 - back >= 0:
        cases.append(T - 2 - back)              # just outside
    W = mixer_weights(layer)
    steps = [[(0, 0, T - rows)], [(0, T - rows, rows)]]
    for hot in cases:
        h = base.clone()
        h[hot, 1] = 3.0
        cache = mod.state_tensors(64, 16, 1, device)
        got = run_mixer(layer, {0: h}, steps, device, cache)[0][T - rows:]
        held = oracle.latents(h.double(), W, "", m, 1e-4)

        def full(c):
            return oracle.latent_attention_mixer(
                h[T - rows:].double(), W, "", m, 1e-4, (c, held[1]),
                pos0=T - rows)

        want = full(held[0])
        assert rel_err(got, want) < TOL
        c2 = held[0].clone()
        c2[hot] = 0                   # without it the last row is different
        moved = row_err(full(c2)[-1:], want[-1:])[0]
        assert (moved > 0.2) == (hot == cases[0])


def attention_layer(device, H, G, D, V, rot, v_mix=False, seed=0, width=40,
                    scale=0.3, scaling=(3.0, 1.5, 5.0, 40.0)):
    m = attention_cfg(H, G, D, V, rot, 150.0, scale, v_mix, scaling)
    f, lo, hi, orig = scaling or (1.0, 1.0, 1.0, 0.0)
    layer, g = one_layer(NormedHeadAttention(NormedHeadAttentionConfig(
        heads=H, kv_heads=G, dim=D, vdim=V, scale=scale, rot_dims=rot,
        rot_base=150.0, rot_factor=f, rot_low=lo, rot_high=hi,
        rot_original=orig, one_in_denominator=True, v_mix=v_mix), width,
        1e-4, torch.float32), width, device, seed)
    mod = layer.mixer
    for p in (mod.q_norm, mod.k_norm):
        p.data.copy_(torch.rand(D, generator=g) + 0.5)
    layer.in_proj.bias.data.copy_(
        torch.randn(layer.in_proj.bias.shape, generator=g) * 0.5)
    mod.o_bias.data.copy_(torch.randn(width, generator=g) * 0.5)
    if v_mix:
        mod.vmix.data.fill_(0.3)
    return layer, m, g


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("H,G,D,V,rot", [
    (6, 2, 10, 7, 6), (1, 1, 4, 4, 4), (4, 4, 64, 64, 32), (8, 1, 9, 20, 2),
    (2, 1, 80, 48, 40), (4, 2, 128, 128, 128), (3, 3, 5, 1, 0),
    (10, 1, 16, 130, 16)])
def test_attention_with_blended_values(device, H, G, D, V, rot):
    """The first layer keeps its own values, a later one blends them in;
    both through mixed steps."""
    layer, m, g = attention_layer(device, H, G, D, V, rot, v_mix=True)
    h = {0: torch.randn(40, 40, generator=g),
         1: torch.randn(25, 40, generator=g)}
    first = {s: torch.randn(v.shape[0], G * V, generator=g)
             for s, v in h.items()}
    W = mixer_weights(layer)
    for shared in (None, first):
        cache = layer.mixer.state_tensors(128, 16, 2, device)
        got = run_mixer(layer, h, MIXED_STEPS, device, cache, shared)
        for s in h:
            x = h[s].double()
            v = oracle.attention_values(
                x, W, "", shared[s].double() if shared else None)
            want = oracle.attention_mixer(
                x, W, "", m, 1e-4, oracle.attention_keys(x, W, "", m, 1e-4),
                v)
            assert rel_err(got[s], want) < TOL, s


@pytest.mark.parametrize("device,D,V", [
    ("cpu", 20, 9)] + [pytest.param("cuda", D, V, marks=pytest.mark.gpu)
                       for D, V in ((20, 9), (64, 64), (128, 128),
                                    (112, 96))])
@pytest.mark.parametrize("hot", [0, 15, 16, 63, 64, 127, 128, 255, 256, 290])
@pytest.mark.parametrize("rows", [1, 2, 43])
def test_far_key_decides_the_row(device, D, V, hot, rows):
    """All queries and one key share a strong direction that does not turn;
    the key sits at page (16), key-tile (64), row-tile (128) and span (256)
    borders of a shuffled context. All other scores are far below the 1 of
    the denominator."""
    H, G, T, rot = 4, 2, 300, 8
    layer, m, g = attention_layer(device, H, G, D, V, rot, scale=1.0)
    a, na = layer.in_proj_rows("q")
    b, nb = layer.in_proj_rows("k")
    w, bias = layer.in_proj.weight.data, layer.in_proj.bias.data
    w[a:a + na] *= 0.05
    w[b:b + nb] *= 0.05
    bias[a:a + na] *= 0.05
    bias[b:b + nb] *= 0.05
    for hh in range(H):
        bias[a + hh * D + rot] = 6.0        # not a turning entry
    for gg in range(G):
        w[b + gg * D + rot, 0] = 6.0
    h = torch.randn(T, 40, generator=g)
    h[:, 0] = -1.0
    h[hot, 0] = 1.0
    steps = [[(0, 0, T - rows)], [(0, T - rows, rows)]]
    cache = layer.mixer.state_tensors(64, 16, 1, device)
    got = run_mixer(layer, {0: h}, steps, device, cache)[0][T - rows:]
    W = mixer_weights(layer)
    x = h.double()
    k = oracle.attention_keys(x, W, "", m, 1e-4)
    v = oracle.attention_values(x, W, "")
    full = lambda kk: oracle.attention_mixer(
        x[T - rows:], W, "", m, 1e-4, kk, v, pos0=T - rows)
    want = full(k)
    assert rel_err(got, want) < TOL
    k2 = k.clone()
    k2[hot] = -k2[hot]
    lost = full(k2)
    assert row_err(lost[-1:], want[-1:])[0] > 0.2
    # with no key in sight the 1 takes all the weight: only the bias is left
    assert rel_err(lost[-1:], W["o.b"][None]) < 0.05


def scan_layer(device, inner, N, R, taps, seed=0, width=40):
    layer, g = one_layer(SelectiveScanMixer(
        SelectiveScanConfig(inner, N, R, taps), width, 1e-4, torch.float32),
        width, device, seed)
    mod = layer.mixer
    mod.conv_b.data.copy_(torch.randn(inner, generator=g) * 0.3)
    mod.dt_bias.data.copy_(torch.rand(inner, generator=g) * 4 - 4)
    mod.a_log.data.copy_(torch.rand(inner, N, generator=g) * 3 - 1.5)
    mod.d_skip.data.copy_(torch.randn(inner, generator=g))
    return layer, scan_cfg(inner, N, R, taps), g


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("inner,N,R,taps", [
    (36, 5, 3, 3), (1, 1, 1, 1), (64, 16, 4, 4), (70, 8, 2, 2),
    (300, 2, 5, 4), (20, 28, 20, 5), (33, 40, 1, 9), (12, 100, 3, 4),
    (9, 256, 2, 1), (128, 4, 2, 4)])
def test_selective_scan_mixer(device, inner, N, R, taps):
    """Portions, two-row portions and decoded rows, with leftovers of
    earlier owners in the slots; a portion long enough to be cut into
    segments."""
    layer, m, g = scan_layer(device, inner, N, R, taps)
    h = {0: torch.randn(40, 40, generator=g) * 2,
         1: torch.randn(25, 40, generator=g) * 2,
         2: torch.randn(523, 40, generator=g) * 2}
    cache = layer.mixer.state_tensors(1, 16, 3, device)
    for v in cache.values():
        v.normal_()
    steps = MIXED_STEPS + [[(2, 0, 31)], [(2, 31, 2)], [(2, 33, 1)],
                           [(2, 34, 1)], [(2, 35, 16)], [(2, 51, 400)],
                           [(2, 451, 33)], [(2, 484, 39)]]
    got = run_mixer(layer, h, steps, device, cache)
    W = mixer_weights(layer)
    for s in h:
        want = oracle.scan_mixer(h[s].double(), W, "", m)
        assert rel_err(got[s], want) < TOL, s


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("C,taps", [(8, 1), (12, 2), (8, 3), (260, 4),
                                    (7, 4), (8, 6)])
@pytest.mark.parametrize("lens", [[500, 3, 2, 531, 1, 1], [9, 2, 1]])
def test_convolution_over_groups(device, C, taps, lens):
    """Groups of unequal length side by side (in runs of rows that cross
    their borders when there are many), each with inputs of an earlier step
    behind it, then one decoded row each; a wide row's column slice."""
    g = torch.Generator().manual_seed(C + taps)
    S = len(lens)
    first = [2 + s % 3 for s in range(S)]
    seqs = [torch.randn(first[s] + n + 1, C + 3, generator=g)
            for s, n in enumerate(lens)]
    w, b = torch.randn(C, taps, generator=g), torch.randn(C, generator=g)
    tail = torch.randn(S, max(taps - 1, 1), C, generator=g).to(device)
    got = [[] for _ in lens]
    a = [0] * S
    for count in (first, lens, [1] * S):
        x = torch.cat([q[a[s]:a[s] + count[s]] for s, q in enumerate(seqs)])
        cu, pos, rows = [0], [], []
        for s in range(S):
            cu.append(cu[-1] + count[s])
            pos += list(range(a[s], a[s] + count[s]))
            rows += [s] * count[s]
        y = seqmix.causal_conv_silu(
            x.to(device)[:, :C], w.to(device), b.to(device), tail,
            mk(cu, device), mk(rows, device), mk(list(range(S)), device),
            mk(pos, device), max_rows=max(count)).cpu()
        for s in range(S):
            got[s].append(y[cu[s]:cu[s + 1]])
            a[s] += count[s]
    for s, q in enumerate(seqs):
        want = oracle.silu(oracle.causal_conv(q[:, :C].double(), w.double(),
                                              b.double()))
        assert torch.allclose(torch.cat(got[s]).double(), want, atol=1e-4)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("lens", [[500, 2, 1, 1], [390, 385], [1100], [2]])
def test_scan_segments_of_unequal_groups(device, lens):
    """The recurrence alone: groups of unequal length side by side (cut
    into segments on the GPU where that fills the chip), continued from a
    state that was left at another length, next to one-row groups."""
    W_, N = 40, 6
    g = torch.Generator().manual_seed(sum(lens))
    T, S = sum(lens), len(lens)
    pre = [3 + s for s in range(S)]           # rows before this step
    seqs = [dict(u=torch.randn(pre[s] + lens[s], W_, generator=g),
                 dt=torch.randn(pre[s] + lens[s], W_, generator=g) - 1,
                 B=torch.randn(pre[s] + lens[s], N, generator=g),
                 C=torch.randn(pre[s] + lens[s], N, generator=g),
                 z=torch.randn(pre[s] + lens[s], W_, generator=g))
            for s in range(S)]
    bias, D = torch.randn(W_, generator=g), torch.randn(W_, generator=g)
    a_log = torch.rand(W_, N, generator=g) * 3 - 3
    state = torch.randn(S, W_, N, generator=g).to(device)

    def step(first, count):
        rows = lambda k: torch.cat([q[k][first[s]:first[s] + count[s]]
                                    for s, q in enumerate(seqs)]).to(device)
        cu = [0]
        pos = []
        for s in range(S):
            cu.append(cu[-1] + count[s])
            pos += list(range(first[s], first[s] + count[s]))
        spans = [(n, 0, None) for n in count if n > 1]
        return seqmix.selective_scan(
            rows("u"), rows("dt"), bias.to(device), a_log.to(device),
            rows("B"), rows("C"), D.to(device), rows("z"), state,
            mk(cu, device), mk(list(range(S)), device), mk(pos, device),
            prefill_spans=spans).cpu()

    step([0] * S, pre)
    got = step(pre, lens)
    a = 0
    for s, q in enumerate(seqs):
        q = {k: v.double() for k, v in q.items()}
        want = oracle.selective_scan(
            q["u"], oracle.softplus(q["dt"] + bias.double()),
            -torch.exp(a_log.double()), q["B"], q["C"], D.double())
        want = (want * oracle.silu(q["z"]))[pre[s]:]
        assert rel_err(got[a:a + lens[s]], want) < TOL, s
        a += lens[s]


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("hot", [0, 1, 31, 32, 63, 127, 128, 255])
@pytest.mark.parametrize("tail", [1, 2, 70])
def test_far_token_is_remembered(device, hot, tail):
    """One token writes a large input and hardly anything decays: it must
    show hundreds of rows later, wherever it sits in a block or segment."""
    T, W_, N = 520, 24, 7
    g = torch.Generator().manual_seed(hot)
    u = torch.randn(T, W_, generator=g) * 0.05
    u[hot] += 30.0
    dt, z = torch.full((T, W_), -3.0), torch.ones(T, W_)
    B = torch.rand(T, N, generator=g) + 0.5
    C = torch.rand(T, N, generator=g) + 0.5
    bias, D = torch.zeros(W_), torch.ones(W_)
    a_log = torch.full((W_, N), -4.0) + torch.rand(W_, N, generator=g)
    state = torch.zeros(1, W_, N, device=device)
    out = []
    cuts = [0, T - tail, T]
    for a, b in zip(cuts, cuts[1:]):
        d = lambda x: x[a:b].contiguous().to(device)
        out.append(seqmix.selective_scan(
            d(u), d(dt), bias.to(device), a_log.to(device), d(B), d(C),
            D.to(device), d(z), state, mk([0, b - a], device),
            mk([0], device), mk(list(range(a, b)), device),
            prefill_spans=[(b - a, b, None)] if b - a > 1 else None).cpu())

    def full(x):
        y = oracle.selective_scan(
            x, oracle.softplus(dt.double()), -torch.exp(a_log.double()),
            B.double(), C.double(), D.double())
        return y * oracle.silu(z.double())

    want = full(u.double())
    got = torch.cat(out)
    assert rel_err(got, want) < TOL
    u2 = u.double().clone()
    u2[hot] = 0
    gap = (full(u2)[-1] - want[-1]).abs().mean() / want[-1].abs().mean()
    assert gap > 0.5


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
    rows = stacked(got["a"], len(toks))
    assert rel_err(rows, want) < TOL
    assert rel_err(rows[:3], want[:3]) < TOL
    assert len(trace) == len(layers) == len(raw["layers"])
    for got_x, want_x in zip(trace, layers):
        assert rel_err(got_x, want_x) < TOL
    one = run_schedule(eng, [[("b", toks[:1], [0])], [("end", "b")]])
    assert rel_err(one["b"][0][None], want[:1]) < TOL


def test_prefill_against_token_by_token_decoding(small):
    raw, eng, W, toks, want, _ = small
    steps = [[("d", [t], [0])] for t in toks]
    steps.append([("end", "d")])
    got = run_schedule(eng, steps)
    assert rel_err(stacked(got["d"], len(toks)), want) < TOL


@pytest.mark.parametrize("expand", [0, 64, 1 << 30])
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
    assert rel_err(stacked(got["p"], len(toks)), want) < TOL


@pytest.mark.parametrize("expand", [0, 1 << 30])
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
        assert rel_err(stacked(got[k], len(v)), ref[k]) < TOL, k
    assert (eng.block_manager.num_free(),
            eng.state_manager.num_free()) == free_before


def test_slot_and_pages_reused_by_a_shorter_request(small):
    """A long request leaves its state and pages behind; the next one in
    the same slot and pages must start from nothing, and one that is left
    out of a step must find its own again."""
    raw, eng, W, toks, want, _ = small
    run_schedule(eng, [[("x", tokens(60, 9), [])], [("end", "x")]])
    got = run_schedule(eng, [[("y", toks[:2], [0, 1])],
                             [("z", tokens(5, 8), [])],
                             [("y", toks[2:9], list(range(7)))],
                             [("end", "y"), ("end", "z")]])
    assert rel_err(stacked(got["y"], 9), want[:9]) < TOL


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
def test_long_decoding_past_windows_pages_and_spans(device):
    raw = {
        "architecture": "Vatunex", "vocab": 50, "width": 32,
        "norm": {"eps": 1e-5},
        "layers": [
            attn(attention_cfg(2, 1, 8, 8, 8, 100.0, 0.35), 16),
            latent(latent_cfg(heads=2, dim=8, rot_dim=8, vdim=16, kv_rank=24,
                              q_rank=12, scale=0.3, window=33), 16),
            scan(scan_cfg(32, 4, 2, 4), 16),
            attn(attention_cfg(4, 1, 6, 8, 2, 100.0, 0.35), None),
        ],
    }
    eng, W = make_engine(raw, device, blocks=24)
    toks = tokens(300, 21, vocab=50)
    want = oracle.forward(toks, W, raw)
    steps = [[("a", toks[:10], list(range(10)))]]
    steps += [[("a", [t], [0])] for t in toks[10:]]
    got = run_schedule(eng, steps)
    assert rel_err(stacked(got["a"], len(toks)), want) < TOL


@pytest.mark.parametrize("device", DEVICES)
def test_values_that_could_hide_faults(device):
    """Single heads, sizes of one, a window of one and none at all, no
    rotation, no stretching, a stretching that touches every or no pair,
    nothing blended, one tap, one state, no feed-forward at all, more value
    than key entries, recurrences only."""
    toks = tokens(24, 7, vocab=31)
    base = {"architecture": "Vatunex", "vocab": 31, "width": 16,
            "norm": {"eps": 1e-6}}
    variants = [
        [latent(latent_cfg(1, 4, 2, 4, 1, 1, 1.0, window=1), 8)],
        [scan(scan_cfg(1, 1, 1, 1), 1), scan(scan_cfg(16, 16, 16, 4), None)],
        [attn(attention_cfg(1, 1, 2, 5, 2, 10.0, 1.0, True, None), None),
         attn(attention_cfg(5, 5, 3, 1, 0, 10.0, 0.5, True,
                            (4.0, 1.0, 4.0, 1e-3)), 4)],
        [latent(latent_cfg(2, 4, 8, 4, 8, 8, 0.5, window=0), 8),
         attn(attention_cfg(4, 2, 8, 4, 4, 10.0, 0.5, False,
                            (4.0, 1.0, 4.0, 1e6)), 8),
         attn(attention_cfg(2, 2, 4, 4, 4, 10.0, 0.5, True), 8)],
        [attn(attention_cfg(2, 1, 4, 8, 2, 10.0, 0.5, True), 8),
         scan(scan_cfg(8, 3, 1, 2), 8),
         attn(attention_cfg(8, 2, 6, 4, 6, 10.0, 0.5, True), None),
         latent(latent_cfg(1, 1, 2, 1, 2, 3, 0.9, window=500), 8)],
    ]
    # the two blended layers of a variant need equal value rows
    variants[2][1] = attn(attention_cfg(5, 5, 3, 1, 0, 10.0, 0.5, True,
                                        (4.0, 1.0, 4.0, 1e-3)), 4)
    for i, layers in enumerate(variants):
        raw = dict(base, layers=layers)
        eng, W = make_engine(raw, device, blocks=8, seed=i)
        want = oracle.forward(toks, W, raw)
        got = run_schedule(eng, [[("a", toks[:2], [0, 1])],
                                 [("a", toks[2:19], list(range(17)))],
                                 [("a", toks[19:20], [0])],
                                 [("a", toks[20:], list(range(4)))]])
        assert rel_err(stacked(got["a"], len(toks)), want) < TOL, i


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

    refused(set_(["layers", 2, "mixer", "kv_heads"], 4))    # 6 heads
    refused(set_(["layers", 2, "mixer", "rot", "dims"], 5))
    refused(set_(["layers", 2, "mixer", "rot", "dims"], 12))
    refused(set_(["layers", 6, "mixer", "vdim"], 13))       # blended rows
    refused(set_(["layers", 1, "mixer", "rot_dim"], 5))
    refused(set_(["layers", 1, "mixer", "mask", "size"], -2))
    refused(set_(["layers", 0, "mixer", "conv"], 0))
    refused(set_(["layers", 0, "mixer", "state"], 0))
    refused(set_(["layers", 1, "type"], "convolution"))
    refused(set_(["layers", 0, "mlp", "kind"], "sparse"))
    refused(set_(["layers"], []))


def test_cache_and_state_declarations():
    raw = small_config()
    eng, _ = make_engine(raw, "cpu", blocks=8)
    caches = eng.runner.kv_caches
    assert caches[0]["ssm"].shape == (4, 36, 5)
    assert caches[0]["conv"].shape == (4, 2, 36)
    assert caches[1]["kv"].shape == (8, 1, 16, 18)
    assert caches[2]["k"].shape == (8, 2, 16, 10)
    assert caches[2]["v"].shape == (8, 2, 16, 7)
    assert caches[5]["ssm"].dtype == torch.float32
    assert eng.runner.model.kv_block_bytes(16) == 16 * 4 * (
        18 + 2 * 17 + 27 + 4 * 11 + 23)


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
    assert mc.architecture == "Vatunex" and mc.model_path == path
    assert registry.required_extensions(mc) == ("seqmix",)
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
    assert rel_err(stacked(got["a"], 20), oracle.forward(toks, Wb, raw)) < TOL
    # a checkpoint that lacks a tensor, or holds an unknown one, is refused
    from safetensors.torch import load_file, save_file

    t = load_file(os.path.join(path, "model.safetensors"))
    held = t.pop("l2.norm1b")
    save_file(t, os.path.join(path, "model.safetensors"))
    with pytest.raises(ValueError):
        LLMEngine(cfg, device="cpu")
    t["l2.norm1b"] = held
    t["l3.norm2"] = held.clone()      # this layer has no feed-forward
    save_file(t, os.path.join(path, "model.safetensors"))
    LLMEngine(cfg, device="cpu")
    t["l4.mix.vmix"] = t["l2.mix.vmix"].clone()   # nothing is blended there
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


@pytest.mark.parametrize("device", DEVICES)
def test_bf16_mode_stays_close_to_oracle(device):
    raw = small_config()
    eng, W = make_engine(raw, device, dtype="bfloat16", seed=2)
    toks = tokens(40, 5)
    want = oracle.forward(toks, W, raw)
    got = run_schedule(eng, [[("a", toks[:17], list(range(17)))],
                             [("a", toks[17:], list(range(23)))]])
    assert row_err(stacked(got["a"], 40), want).median() < 0.05


# ------------------------------------------------------------- GPU only

def tiled_config():
    """Sizes with MFMA tile kernels in both forms of latent attention and
    in the attention layers."""
    big = dict(dim=32, rot_dim=32, vdim=64, kv_rank=256, q_rank=48,
               scale=0.125, window=150)
    return {
        "architecture": "Vatunex", "vocab": 300, "width": 128,
        "norm": {"eps": 1e-5},
        "layers": [
            latent(latent_cfg(heads=4, **big), 192),
            attn(attention_cfg(4, 2, 64, 64, 32, 1e4, 0.125), 192),
            scan(scan_cfg(256, 16, 8, 4), 192),
            attn(attention_cfg(2, 1, 128, 128, 96, 1e4, 0.09, v_mix=True),
                 192),
            latent(latent_cfg(heads=2, **dict(big, dim=96, vdim=128,
                                              window=77)), 192),
        ],
    }


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("expand", [0, 64, 1 << 30])
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
