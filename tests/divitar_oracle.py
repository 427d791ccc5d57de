"""Plain whole-sequence Divitar in float64: the oracle of tests/test_divitar.py.

One function per mechanism, written from the design's equations (the notation is that of the
model's docstring in ``dgi/models/divitar.py``); no cache, no batching, no state carried between
calls and no code shared with the product path.  ``P`` is a dict name -> float64 tensor in the
checkpoint naming (``l<i>.mix.q`` ...), ``cfg`` the parsed ``config.json`` dictionary.  Keys and
values are formed explicitly per head and every query takes its visible keys by an explicit slice.
"""
import math

import torch

F = torch.float64


def gelu_tanh(z):
    return 0.5 * z * (1 + torch.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z ** 3)))


def silu(z):
    return z * torch.sigmoid(z)


def relu_squared(z):
    return torch.where(z > 0, z * z, torch.zeros_like(z))


def unit_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def rms_norm(x, w, eps):
    return unit_rms(x, eps) * w


def linear_freqs(rot):
    """Angular frequency of every rotary pair, all divided by the scaling factor."""
    d, base = int(rot["dims"]), float(rot["base"])
    factor = float((rot.get("scaling") or {}).get("factor", 1.0))
    return [base ** (-2.0 * i / d) / factor for i in range(d // 2)]


def ramp_freqs(rot):
    """(frequency of every pair, factor on cos and sin) of the ramp form: slow pairs are divided by the
    scaling factor, fast ones stay, those between are blended."""
    d, base = int(rot["dims"]), float(rot["base"])
    plain = [base ** (-2.0 * i / d) for i in range(d // 2)]
    s = rot.get("scaling")
    if not s:
        return plain, 1.0
    factor, orig = float(s["factor"]), float(s["original"])

    def pair_at(turns):
        return d * math.log(orig / (2 * math.pi * turns)) / (2 * math.log(base))

    lo = max(math.floor(pair_at(float(s["fast"]))), 0)
    hi = min(math.ceil(pair_at(float(s["slow"]))), d - 1)
    out = []
    for i, f in enumerate(plain):
        r = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(f / factor * r + f * (1 - r))
    return out, 0.1 * math.log(factor) + 1.0


def rotate_halves(v, pos, rot):
    """Rotary position of the vector ``v``: pairs (i, i + dims / 2) of its first ``dims`` entries."""
    out = v.clone()
    half = int(rot["dims"]) // 2
    for i, f in enumerate(linear_freqs(rot)):
        c, s = math.cos(pos * f), math.sin(pos * f)
        out[i] = v[i] * c - v[i + half] * s
        out[i + half] = v[i + half] * c + v[i] * s
    return out


def rotate_pairs(v, pos, rot):
    """Rotary position of the vector ``v``: pairs (2 i, 2 i + 1) of its first ``dims`` entries."""
    out = v.clone()
    fs, stretch = ramp_freqs(rot)
    for i, f in enumerate(fs):
        c, s = stretch * math.cos(pos * f), stretch * math.sin(pos * f)
        out[2 * i] = v[2 * i] * c - v[2 * i + 1] * s
        out[2 * i + 1] = v[2 * i + 1] * c + v[2 * i] * s
    return out


def chunk_start(i, size):
    """First key that position ``i`` sees when a sequence is cut into chunks of ``size`` positions."""
    return (i // size) * size if size else 0


def window_start(i, size):
    """First key that position ``i`` sees when it sees the last ``size`` positions, itself included."""
    return max(0, i - size + 1) if size else 0


def attention(P, pre, m, h):
    """Grouped-query attention whose values are the unrotated keys, chunked, one output gate per head."""
    T = h.shape[0]
    H, G, d = int(m["heads"]), int(m["kv_heads"]), int(m["dim"])
    q = (h @ P[pre + "mix.q"].T + P[pre + "mix.q.b"]).view(T, H, d)
    k = (h @ P[pre + "mix.k"].T + P[pre + "mix.k.b"]).view(T, G, d)
    g = torch.sigmoid(h @ P[pre + "mix.g"].T)
    kr = torch.stack([torch.stack([rotate_halves(k[t, j], t, m["rot"]) for j in range(G)]) for t in range(T)])
    size = int((m.get("mask") or {}).get("size") or 0)
    out = torch.zeros(T, H * d, dtype=F)
    for i in range(T):
        lo = chunk_start(i, size)
        for hh in range(H):
            j = hh // (H // G)
            s = kr[lo:i + 1, j] @ rotate_halves(q[i, hh], i, m["rot"]) * float(m["scale"])
            out[i, hh * d:(hh + 1) * d] = (torch.softmax(s, 0) @ k[lo:i + 1, j]) * g[i, hh]
    return out @ P[pre + "mix.o"].T


def softmax_with_sink(s, sink):
    """Weights of the scores ``s`` when exp(sink) is one more term of the denominator."""
    top = torch.maximum(s.max(), sink)
    e = torch.exp(s - top)
    return e / (e.sum() + torch.exp(sink - top))


def latent_kv(P, pre, m, h, eps):
    """(latent c [T, kv_rank], rotated shared key part [T, rot_dim]) of the layer whose tensors start with ``pre``."""
    r = int(m["kv_rank"])
    d = h @ P[pre + "mix.dkv"].T
    return (rms_norm(d[:, :r], P[pre + "mix.dkv.norm"], eps),
            torch.stack([rotate_pairs(d[t, r:], t, m["rot"]) for t in range(d.shape[0])]))


def latent_attention(P, pre, m, h, eps, shared=None):
    """One latent-attention mixer on the whole sequence ``h`` [T, W]; ``shared`` = (c, r) of the layer named by
    ``kv_from``.  Returns (output, (c, r))."""
    T = h.shape[0]
    H, dn, dr, dv = int(m["heads"]), int(m["dim"]), int(m["rot_dim"]), int(m["vdim"])
    q = (h @ P[pre + "mix.q"].T).view(T, H, dn + dr)
    c, r = shared if shared is not None else latent_kv(P, pre, m, h, eps)
    kn = (c @ P[pre + "mix.uk"].T).view(T, H, dn)
    v = (c @ P[pre + "mix.uv"].T).view(T, H, dv)
    size = int((m.get("mask") or {}).get("size") or 0)
    out = torch.zeros(T, H * dv, dtype=F)
    for i in range(T):
        lo = window_start(i, size)
        for hh in range(H):
            s = (kn[lo:i + 1, hh] @ q[i, hh, :dn] + r[lo:i + 1] @ rotate_pairs(q[i, hh, dn:], i, m["rot"])) * float(m["scale"])
            out[i, hh * dv:(hh + 1) * dv] = softmax_with_sink(s, P[pre + "mix.sink"][hh]) @ v[lo:i + 1, hh]
    return out @ P[pre + "mix.o"].T, (c, r)


def dense_ff(P, pre, h):
    return relu_squared(h @ P[pre + "mlp.up"].T) @ P[pre + "mlp.down"].T


def route(z, top, scale):
    """Chosen experts and their weights from router logits ``z`` [E]: sigmoid scores, the ``top`` largest,
    normalised to a sum of one, times ``scale``."""
    s = torch.sigmoid(z)
    order = sorted(range(z.shape[0]), key=lambda e: (-float(s[e]), e))[:top]
    total = sum(s[e] for e in order) + 1e-20
    return order, [s[e] / total * scale for e in order]


def glu(P, pre, x):
    return (silu(x @ P[pre + ".gate"].T) * (x @ P[pre + ".up"].T)) @ P[pre + ".down"].T


def moe_ff(P, pre, f, h):
    r = f["router"]
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, w in zip(*route(h[t] @ P[pre + "mlp.router"].T, int(r["top"]), float(r["scale"]))):
            out[t] += w * glu(P, f"{pre}mlp.e{e}", h[t])
        if f.get("shared"):
            out[t] += glu(P, pre + "mlp.shared", h[t])
    return out


def token_side(P, cfg, pre, li, x, tokens, eps, mult):
    """Per-layer token input added to the stream after the feed-forward."""
    d = int(cfg["token_side"]["dim"])
    e = P["side.embed"][torch.tensor(tokens)][:, li * d:(li + 1) * d]
    y = (gelu_tanh(x @ P[pre + "side.gate"].T) * e) @ P[pre + "side.proj"].T
    return x + mult * unit_rms(y, eps) * P[pre + "side.norm"]


def forward(P, cfg, tokens, return_layers=False):
    """Logits [T, vocab] of a whole sequence (and the stream after every layer)."""
    eps, mult = float(cfg["norm"]["eps"]), float(cfg.get("residual_mult", 1.0))
    x = P["embed"][torch.tensor(tokens)].clone()
    kept, streams = {}, []
    for li, L in enumerate(cfg["layers"]):
        pre, m, f = f"l{li}.", L["mixer"], L.get("mlp")
        h = rms_norm(x, P[pre + "norm1"], eps)
        if L["type"] == "attention":
            y = attention(P, pre, m, h)
        else:
            src = m.get("kv_from")
            y, kept[li] = latent_attention(P, pre, m, h, eps, None if src is None else kept[int(src)])
        x = x + mult * y
        if f is not None:
            h = rms_norm(x, P[pre + "norm2"], eps)
            x = x + mult * (dense_ff(P, pre, h) if f.get("kind", "dense") == "dense" else moe_ff(P, pre, f, h))
        if cfg.get("token_side"):
            x = token_side(P, cfg, pre, li, x, tokens, eps, mult)
        streams.append(x.clone())
    logits = rms_norm(x, P["final.norm"], eps) @ P["head"].T * float(cfg.get("logit_scale", 1.0))
    return (logits, streams) if return_layers else logits
