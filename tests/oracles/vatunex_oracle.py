"""Plain, slow float64 oracle of the Vatunex design: one function per
mechanism, explicit loops over tokens and heads, no paging, no batching,
no state objects. It shares no code with fusioninfer_amd; tests compare
the engine (CPU ops or HIP kernels) against it.

Weights use the checkpoint naming (``l<i>.mix.dq`` ...), as a dict of
float64 tensors; ``cfg`` is the config.json dict.

The design in short: an RMS norm in front of and behind every sublayer
(weights stored around zero); the mixer is windowed attention over cached
low-rank latents, grouped-query attention with normed heads, half-rotation
with frequencies stretched for long contexts, a one in the softmax
denominator and values blended with those of an earlier layer, or a
selective state-space recurrence behind a short convolution; the
feed-forward is a plain GELU unit.
"""

import math

import torch

F64 = torch.float64


def rms_norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


def centred_norm(x, w, eps):
    """RMS norm whose weight is stored as its distance from one."""
    return rms_norm(x, 1.0 + w, eps)


def silu(z):
    return z / (1.0 + torch.exp(-z))


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(
        math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def softplus(z):
    return torch.clamp(z, min=0) + torch.log1p(torch.exp(-torch.abs(z)))


def dense_mlp(h, W, pre):
    return gelu_tanh(h @ W[pre + "up"].T) @ W[pre + "down"].T


# --------------------------------------------------------------- rotation

def rotary_frequencies(rot):
    """dims/2 angular frequencies; with ``scaling`` long wavelengths are
    stretched by ``factor``, short ones kept, the ones between blended."""
    dims, base = int(rot["dims"]), float(rot["base"])
    out = []
    sc = rot.get("scaling")
    for i in range(dims // 2):
        f = base ** (-2.0 * i / dims)
        if sc:
            turns = float(sc["original"]) * f / (2.0 * math.pi)
            if turns < sc["low"]:
                f = f / sc["factor"]
            elif turns <= sc["high"]:
                s = (turns - sc["low"]) / (sc["high"] - sc["low"])
                f = (1.0 - s) * f / sc["factor"] + s * f
        out.append(f)
    return out


def rotate_half(x, pos, freqs):
    """One vector: entry i turns with entry i + n (n = len(freqs)); entries
    from 2 n on pass."""
    n = len(freqs)
    c = torch.tensor([math.cos(pos * f) for f in freqs], dtype=F64)
    s = torch.tensor([math.sin(pos * f) for f in freqs], dtype=F64)
    u, v = x[:n], x[n:2 * n]
    return torch.cat([u * c - v * s, v * c + u * s, x[2 * n:]])


# -------------------------------------------------------------- attention

def attend(q, k, v, scale, first, window=0, one=False):
    """One head. Row t of q stands at position first + t; k and v hold
    positions 0...; ``window`` 0: every earlier key; ``one``: a further 1 in
    the denominator."""
    out = []
    for t in range(q.shape[0]):
        p = first + t
        lo = max(0, p - window + 1) if window else 0
        s = (k[lo:p + 1] @ q[t]) * scale
        m = s.max()
        if one:
            m = torch.clamp(m, min=0.0)
        e = torch.exp(s - m)
        den = e.sum()
        if one:
            den = den + torch.exp(-m)
        out.append((e / den) @ v[lo:p + 1])
    return torch.stack(out)


def latents(h, W, pre, m, eps):
    """What is kept of every token: (normed latent, rotated key part)."""
    R = m["kv_rank"]
    z = h @ W[pre + "dkv"].T
    freqs = rotary_frequencies(m["rot"])
    c = rms_norm(z[:, :R], W[pre + "dkv.norm"], eps)
    kr = torch.stack([rotate_half(z[t, R:], t, freqs)
                      for t in range(h.shape[0])])
    return c, kr


def latent_attention_mixer(h, W, pre, m, eps, held=None, pos0=0):
    """h: the input rows of positions pos0...; ``held``: the latents of all
    positions up to the last row (default: of h itself)."""
    H, D, V = m["heads"], m["dim"], m["vdim"]
    R = m["rot_dim"]
    c, kr = held if held is not None else latents(h, W, pre, m, eps)
    freqs = rotary_frequencies(m["rot"])
    q = rms_norm(h @ W[pre + "dq"].T, W[pre + "dq.norm"], eps)
    q = q @ W[pre + "uq"].T
    k = c @ W[pre + "uk"].T
    v = c @ W[pre + "uv"].T
    window = int((m.get("mask") or {}).get("size", 0))
    heads = []
    for a in range(H):
        qa = q[:, a * (D + R):(a + 1) * (D + R)].clone()
        for t in range(h.shape[0]):
            qa[t, D:] = rotate_half(qa[t, D:], pos0 + t, freqs)
        ka = torch.cat([k[:, a * D:(a + 1) * D], kr], dim=1)
        heads.append(attend(qa, ka, v[:, a * V:(a + 1) * V], m["scale"],
                            pos0, window))
    return torch.cat(heads, dim=-1) @ W[pre + "o"].T


def mix_values(v, v_first, lam):
    return (1.0 - lam) * v + lam * v_first


def attention_values(h, W, pre, v_first=None):
    """A layer's values, blended with ``v_first`` if there are such."""
    v = h @ W[pre + "v"].T + W[pre + "v.b"]
    if v_first is None:
        return v
    return mix_values(v, v_first, W[pre + "vmix"].reshape(()))


def attention_keys(h, W, pre, m, eps, pos0=0):
    """Normed and rotated keys [T, kv_heads, dim]."""
    D = m["dim"]
    freqs = rotary_frequencies(m["rot"])
    k = h @ W[pre + "k"].T + W[pre + "k.b"]
    out = torch.zeros(h.shape[0], m["kv_heads"], D, dtype=F64)
    for t in range(h.shape[0]):
        for g in range(m["kv_heads"]):
            x = rms_norm(k[t, g * D:(g + 1) * D], W[pre + "k.norm"], eps)
            out[t, g] = rotate_half(x, pos0 + t, freqs)
    return out


def attention_mixer(h, W, pre, m, eps, k, v, pos0=0):
    """h: the rows of positions pos0...; k [*, G, dim] and v [*, G * vdim]:
    keys and values of all positions up to the last row."""
    H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    freqs = rotary_frequencies(m["rot"])
    q = h @ W[pre + "q"].T + W[pre + "q.b"]
    heads = []
    for a in range(H):
        g = a // (H // G)
        qa = torch.stack([
            rotate_half(rms_norm(q[t, a * D:(a + 1) * D],
                                 W[pre + "q.norm"], eps), pos0 + t, freqs)
            for t in range(h.shape[0])])
        heads.append(attend(qa, k[:, g], v[:, g * V:(g + 1) * V],
                            m["scale"], pos0, one=True))
    return torch.cat(heads, dim=-1) @ W[pre + "o"].T + W[pre + "o.b"]


# -------------------------------------------------------- selective scan

def causal_conv(x, w, b):
    """Per channel over time; w [channels, taps], last tap: the token."""
    T, taps = x.shape[0], w.shape[1]
    out = torch.zeros_like(x)
    for t in range(T):
        out[t] = b
        for j in range(taps):
            u = t - (taps - 1) + j
            if u >= 0:
                out[t] = out[t] + w[:, j] * x[u]
    return out


def selective_scan(x, dt, A, B, C, D):
    """x, dt [T, channels]; A [channels, states]; B, C [T, states]."""
    S = torch.zeros_like(A)
    out = []
    for t in range(x.shape[0]):
        S = torch.exp(dt[t][:, None] * A) * S \
            + (dt[t] * x[t])[:, None] * B[t][None, :]
        out.append(S @ C[t] + D * x[t])
    return torch.stack(out)


def scan_mixer(h, W, pre, m):
    inner, N, R = m["inner"], m["state"], m["dt_rank"]
    xz = h @ W[pre + "in"].T
    x, z = xz[:, :inner], xz[:, inner:]
    x = silu(causal_conv(x, W[pre + "conv"], W[pre + "conv.b"]))
    p = x @ W[pre + "x"].T
    dt = softplus(p[:, :R] @ W[pre + "dt"].T + W[pre + "dt.b"])
    y = selective_scan(x, dt, -torch.exp(W[pre + "A_log"]), p[:, R:R + N],
                       p[:, R + N:], W[pre + "D"])
    return (y * silu(z)) @ W[pre + "o"].T


# ------------------------------------------------------------------ model

def forward(tokens, W, cfg, trace=None):
    """Logits [T, vocab] of a whole sequence; ``trace``: a list that gets
    the stream after every layer."""
    eps = cfg["norm"]["eps"]
    x = W["embed"][torch.tensor(tokens)]
    v_first = None
    for i, L in enumerate(cfg["layers"]):
        p = f"l{i}."
        m, pre = L["mixer"], f"l{i}.mix."
        h = centred_norm(x, W[p + "norm1"], eps)
        if L["type"] == "latent_attention":
            y = latent_attention_mixer(h, W, pre, m, eps)
        elif L["type"] == "attention":
            v = attention_values(h, W, pre,
                                 v_first if m.get("v_mix") else None)
            if m.get("v_mix") and v_first is None:
                v_first = v
            y = attention_mixer(h, W, pre, m, eps,
                                attention_keys(h, W, pre, m, eps), v)
        else:
            y = scan_mixer(h, W, pre, m)
        x = x + centred_norm(y, W[p + "norm1b"], eps)
        if L.get("mlp"):
            y = dense_mlp(centred_norm(x, W[p + "norm2"], eps), W, p + "mlp.")
            x = x + centred_norm(y, W[p + "norm2b"], eps)
        if trace is not None:
            trace.append(x.clone())
    return centred_norm(x, W["final.norm"], eps) @ W["head"].T


def greedy(prompt, W, cfg, n):
    toks = list(prompt)
    for _ in range(n):
        toks.append(int(forward(toks, W, cfg)[-1].argmax()))
    return toks[len(prompt):]
