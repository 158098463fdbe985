"""Plain, slow float64 oracle of the Sufavik design: one function per
mechanism, explicit loops over tokens and heads, no paging, no batching,
no state objects. It shares no code with fusioninfer_amd; tests compare
the engine (CPU ops or HIP kernels) against it.

Weights use the checkpoint naming (``l<i>.mix.dq`` ...), as a dict of
float64 tensors; ``cfg`` is the config.json dict.

The design in short: several copies of the stream, all equal to the token
embedding at the start; every sublayer reads a weighted sum of the copies
through an RMS norm, and its result goes back to every copy while the
copies are mixed by a small matrix. The mixer is an attention over cached
low-rank latents (queries through a latent of their own, a rotated part
with blended frequencies, a sigmoid gate per head; a layer may read an
earlier layer's latents) or a matrix memory with exponential gates. The
feed-forward is squared-relu, or routed silu-gated experts of which some
are the identity, next to a gated shared expert.
"""

import math

import torch

F64 = torch.float64


def rms_norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


def silu(z):
    return z / (1.0 + torch.exp(-z))


# ------------------------------------------------------------ stream copies

def read_streams(xs, w_in):
    """Weighted sum of the copies xs [S, T, width]."""
    u = torch.zeros_like(xs[0])
    for s in range(xs.shape[0]):
        u = u + w_in[s] * xs[s]
    return u


def write_streams(xs, y, mix, w_out):
    """New copies: copy t is sum_s mix[s, t] * (old copy s) + w_out[t] * y."""
    new = []
    for t in range(xs.shape[0]):
        acc = w_out[t] * y
        for s in range(xs.shape[0]):
            acc = acc + mix[s, t] * xs[s]
        new.append(acc)
    return torch.stack(new)


# ---------------------------------------------------------- matrix memory

def log_sigmoid(z):
    return -math.log1p(math.exp(-z)) if z > -30 else z


def memory_gates(h, W, pre, m):
    """(log input gate, log forget gate), [T][heads] python floats."""
    cap = float(m["gate_cap"])
    zi = h @ W[pre + "i"].T + W[pre + "i.b"]
    zf = h @ W[pre + "f"].T + W[pre + "f.b"]
    li = [[cap * math.tanh(float(z) / cap) for z in row] for row in zi]
    lf = [[log_sigmoid(cap * math.tanh(float(z) / cap)) for z in row]
          for row in zf]
    return li, lf


def memory_scan(q, k, v, li, lf):
    """One head: q, k [T, dim], v [T, vdim] and per-token log gates; returns
    the read-outs [T, vdim]. Token by token with the running maximum."""
    T, D = q.shape
    S = torch.zeros(D, v.shape[1], dtype=F64)
    n = torch.zeros(D, dtype=F64)
    m = 0.0
    out = []
    for t in range(T):
        m_new = max(lf[t] + m, li[t])
        keep, add = math.exp(lf[t] + m - m_new), math.exp(li[t] - m_new)
        S = keep * S + add * torch.outer(k[t], v[t])
        n = keep * n + add * k[t]
        m = m_new
        den = max(abs(float(n @ q[t])), math.exp(-m)) + 1e-6
        out.append((S.T @ q[t]) / den)
    return torch.stack(out)


def memory_mixer(h, W, pre, m, eps):
    H, D, V = m["heads"], m["dim"], m["vdim"]
    q = (h @ W[pre + "q"].T) * D ** -0.5
    k = h @ W[pre + "k"].T
    v = h @ W[pre + "v"].T
    li, lf = memory_gates(h, W, pre, m)
    heads = []
    for a in range(H):
        o = memory_scan(q[:, a * D:(a + 1) * D], k[:, a * D:(a + 1) * D],
                        v[:, a * V:(a + 1) * V],
                        [r[a] for r in li], [r[a] for r in lf])
        heads.append(rms_norm(o, 1.0, eps))
    o = torch.cat(heads, dim=-1) * W[pre + "norm"]
    return (o * torch.sigmoid(h @ W[pre + "g"].T)) @ W[pre + "o"].T


# -------------------------------------------------------- latent attention

def rotary_frequencies(rot):
    """([dims/2] angular frequencies, factor on cos and sin)."""
    dims, base = int(rot["dims"]), float(rot["base"])
    f = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    sc = rot.get("scaling")
    if not sc:
        return f, 1.0
    factor = float(sc["factor"])

    def pair_with(turns):
        return (dims * math.log(sc["original"] / (2.0 * math.pi * turns))
                / (2.0 * math.log(base)))

    lo = max(math.floor(pair_with(sc["fast"])), 0)
    hi = min(math.ceil(pair_with(sc["slow"])), dims - 1)
    out = []
    for i, fi in enumerate(f):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(fi / factor * ramp + fi * (1.0 - ramp))
    return out, 0.1 * math.log(factor) + 1.0


def rotate(x, pos, freqs, mult):
    """x [..., >= 2 len(freqs)]: neighbours (2i, 2i+1) turn by
    pos * freqs[i]; cos and sin carry ``mult``."""
    y = x.clone()
    for i, f in enumerate(freqs):
        c, s = math.cos(pos * f) * mult, math.sin(pos * f) * mult
        a, b = x[..., 2 * i], x[..., 2 * i + 1]
        y[..., 2 * i] = a * c - b * s
        y[..., 2 * i + 1] = b * c + a * s
    return y


def latents(h, W, pre, m, eps, pos0=0):
    """What is cached of rows h at positions pos0..: the normed latent and
    the rotated shared key part."""
    C = m["kv_rank"]
    z = h @ W[pre + "dkv"].T
    c = rms_norm(z[:, :C], W[pre + "dkv.norm"], eps)
    freqs, mult = rotary_frequencies(m["rot"])
    kr = torch.stack([rotate(z[t, C:], pos0 + t, freqs, mult)
                      for t in range(h.shape[0])])
    return c, kr


def attend_row(qn, qr, kn, kr, v, p, scale):
    """One row: qn [H, dim], qr [H, rot] against the expanded keys
    kn [>=p+1, H, dim], the shared kr [>=p+1, rot] and v [>=p+1, H, vdim]."""
    out = []
    for a in range(qn.shape[0]):
        sc = (kn[:p + 1, a] @ qn[a] + kr[:p + 1] @ qr[a]) * scale
        e = torch.exp(sc - sc.max())
        out.append((e / e.sum()) @ v[:p + 1, a])
    return torch.stack(out)


def latent_attention_mixer(h, W, pre, m, eps, held, pos0=0):
    """h: rows at positions pos0..; held = (latents, rotated key parts) of
    positions 0.. (own or borrowed)."""
    T, H, D, R, V = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    c, kr = held
    cq = rms_norm(h @ W[pre + "dq"].T, W[pre + "dq.norm"], eps)
    q = (cq @ W[pre + "uq"].T).reshape(T, H, D + R)
    kn = (c @ W[pre + "uk"].T).reshape(-1, H, D)
    v = (c @ W[pre + "uv"].T).reshape(-1, H, V)
    freqs, mult = rotary_frequencies(m["rot"])
    gate = torch.sigmoid(h @ W[pre + "g"].T)
    rows = []
    for t in range(T):
        qr = rotate(q[t, :, D:], pos0 + t, freqs, mult)
        o = attend_row(q[t, :, :D], qr, kn, kr, v, pos0 + t, m["scale"])
        rows.append((o * gate[t][:, None]).reshape(-1))
    return torch.stack(rows) @ W[pre + "o"].T


# ------------------------------------------------------------ feed-forward

def squared_relu_unit(h, W, pre):
    return torch.relu(h @ W[pre + "up"].T) ** 2 @ W[pre + "down"].T


def gated_unit(h, W, pre):
    return (silu(h @ W[pre + "gate"].T) * (h @ W[pre + "up"].T)) \
        @ W[pre + "down"].T


def route(z, correction, top):
    """z: logits of ONE token over experts and identity experts. Returns
    [(index, weight)]."""
    e = torch.exp(z - z.max())
    s = e / e.sum()
    c = s + correction
    order = sorted(range(len(c)), key=lambda a: (-float(c[a]), a))
    return [(a, s[a]) for a in order[:top]]


def routed_experts(h, W, pre, mlp):
    n = mlp["router"]["experts"]
    rows = []
    for t in range(h.shape[0]):
        acc = torch.zeros_like(h[t])
        for e, w in route(W[pre + "router"] @ h[t], W[pre + "correction"],
                          mlp["router"]["top"]):
            acc = acc + w * (h[t] if e >= n else
                             gated_unit(h[t:t + 1], W, f"{pre}e{e}.")[0])
        rows.append(acc)
    out = torch.stack(rows)
    if mlp.get("shared"):
        gate = torch.sigmoid(h @ W[pre + "shared.sg"].T)
        out = out + gate * gated_unit(h, W, pre + "shared.")
    return out


def feed_forward(h, W, pre, mlp):
    if mlp["kind"] == "dense":
        return squared_relu_unit(h, W, pre)
    return routed_experts(h, W, pre, mlp)


# ------------------------------------------------------------------- model

def forward(tokens, W, cfg, trace=None):
    """Whole sequence from position 0; returns logits [T, vocab]. ``trace``:
    list that receives the sum of the copies after every layer."""
    eps = cfg["norm"]["eps"]
    x = W["embed"][torch.as_tensor(list(tokens), dtype=torch.long)]
    xs = torch.stack([x.clone() for _ in range(cfg["streams"])])
    held = {}
    for i, L in enumerate(cfg["layers"]):
        p = f"l{i}."
        m = L["mixer"]

        def mixer(h):
            if L["type"] == "mlstm":
                return memory_mixer(h, W, p + "mix.", m, eps)
            src = m.get("kv_from")
            if src is None:
                held[i] = latents(h, W, p + "mix.", m, eps)
                src = i
            return latent_attention_mixer(h, W, p + "mix.", m, eps, held[src])

        def ff(h):
            return feed_forward(h, W, p + "mlp.", L["mlp"])

        for q, sub in ((1, mixer), (2, ff)):
            if q == 2 and not L.get("mlp"):
                continue
            u = read_streams(xs, W[f"{p}hc{q}.in"])
            y = sub(rms_norm(u, W[f"{p}norm{q}"], eps))
            xs = write_streams(xs, y, W[f"{p}hc{q}.mix"], W[f"{p}hc{q}.out"])
        if trace is not None:
            trace.append(xs.sum(0))
    return rms_norm(xs.sum(0), W["final.norm"], eps) @ W["head"].T


def greedy(prompt, W, cfg, n_new):
    toks = list(prompt)
    for _ in range(n_new):
        toks.append(int(forward(toks, W, cfg)[-1].argmax()))
    return toks[len(prompt):]
