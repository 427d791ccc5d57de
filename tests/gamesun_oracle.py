"""Plain float64 Gamesun: whole sequences, one function per mechanism.

Nothing here is shared with ``dgi``: no cache, no state slots, no batching, no kernels.  A model
is (``cfg``, ``w``): the dictionary of the design's ``config.json`` and a name -> float64 tensor
map with the checkpoint's tensor names.  ``forward`` returns the logits of every position and,
on request, the residual stream after every layer.

Notation: W width, T tokens, h the mixer's normed input, rms(v) = sqrt(mean(v^2) + eps).
"""
from __future__ import annotations

import torch

F64 = torch.float64


def rms_unit(v, eps):
    return v / torch.sqrt((v * v).mean(-1, keepdim=True) + eps)


def silu(z):
    return z * torch.sigmoid(z)


def lin(w, x):
    return x @ w.T


# ------------------------------------------------------------------ embedding
def position_vector(p: int, W: int):
    """sin / cos interleaved: entry 2i sin(p f_i), entry 2i + 1 cos(p f_i), f_i = 10000^(-2i / W)."""
    out = torch.zeros(W, dtype=F64)
    for c in range(W):
        a = torch.tensor(float(p), dtype=F64) * 10000.0 ** (-2.0 * (c // 2) / W)
        out[c] = torch.sin(a) if c % 2 == 0 else torch.cos(a)
    return out


def embed(w, tokens, scale):
    W = w["embed"].shape[1]
    return torch.stack([w["embed"][t] * scale + position_vector(p, W) for p, t in enumerate(tokens)], 0)


# ------------------------------------------------------------------ attention
def raw_scores(q, k):
    """q [T, H, d], k [T, G, d] -> q . k per query head [H, T, T] (query i, key j)."""
    H, G = q.shape[1], k.shape[1]
    return torch.stack([q[:, h] @ k[:, h // (H // G)].T for h in range(H)], 0)


def window_mask(T: int, window: int):
    """True where query i may see key j: 0 <= i - j < window (0: every earlier key)."""
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    ok = j <= i
    return ok & (i - j < window) if window else ok


def talk_sigmoid_attention(q, k, v, scale, talk, pb, window):
    """Scores mixed over heads, then an independent sigmoid weight per key: [T, H, dv]."""
    H, G = q.shape[1], v.shape[1]
    s = torch.einsum("hg,gij->hij", talk, raw_scores(q, k) * scale)
    p = torch.sigmoid(s + pb[:, None, None]) * window_mask(q.shape[0], window)
    return torch.stack([p[h] @ v[:, h // (H // G)] for h in range(H)], 1)


def temp_softmax_attention(q, k, v, scale, temp, window):
    """Softmax over the visible keys of scores times a number per head: [T, H, dv]."""
    H, G = q.shape[1], v.shape[1]
    s = raw_scores(q, k) * scale * temp[:, None, None]
    s = s.masked_fill(~window_mask(q.shape[0], window), -float("inf"))
    p = torch.softmax(s, -1)
    return torch.stack([p[h] @ v[:, h // (H // G)] for h in range(H)], 1)


# ------------------------------------------------------------------ recurrences
def channel_decay(z, tau):
    """sigmoid(z)^(1 / tau)."""
    return torch.sigmoid(z) ** (1.0 / tau)


def gated_linear_core(q, k, v, dec):
    """S <- diag(dec) S + k v^T, o = S^T q; q, k, dec [T, H, D], v [T, H, V] -> [T, H, V]."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[2], dtype=F64)
    out = torch.zeros(T, H, v.shape[2], dtype=F64)
    for t in range(T):
        S = dec[t, :, :, None] * S + k[t, :, :, None] * v[t, :, None, :]
        out[t] = torch.einsum("hkv,hk->hv", S, q[t])
    return out


def lightning_core(q, k, v, dec):
    """S <- dec_h S + k v^T, o = S^T q; dec [H]."""
    T, H, D = q.shape
    return gated_linear_core(q, k, v, dec[None, :, None].expand(T, H, D))


# ------------------------------------------------------------------ mixers
def heads(x, n):
    return x.view(x.shape[0], n, -1)


def proj(w, name, x):
    y = lin(w[name], x)
    return y + w[name + ".b"] if name + ".b" in w else y


def left_talk(w, p, m, h):
    H, G = int(m["heads"]), int(m["kv_heads"])
    o = talk_sigmoid_attention(heads(proj(w, p + "q", h), H), heads(proj(w, p + "k", h), G), heads(proj(w, p + "v", h), G),
                               float(m["scale"]), w[p + "talk"], w[p + "pb"], int((m.get("mask") or {}).get("size") or 0))
    return proj(w, p + "o", o.reshape(h.shape[0], -1))


def left_softmax(w, p, m, h):
    H, G = int(m["heads"]), int(m["kv_heads"])
    o = temp_softmax_attention(heads(lin(w[p + "q"], h), H), heads(lin(w[p + "k"], h), G), heads(lin(w[p + "v"], h), G),
                               float(m["scale"]), w[p + "temp"], int((m.get("mask") or {}).get("size") or 0))
    return lin(w[p + "o"], o.reshape(h.shape[0], -1))


def right_gated(w, p, m, h, eps):
    H, D = int(m["heads"]), int(m["dim"])
    dec = channel_decay(lin(w[p + "a2"], lin(w[p + "a1"], h)) + w[p + "a2.b"], float(m["tau"]))
    o = gated_linear_core(heads(lin(w[p + "q"], h), H) * D ** -0.5, heads(lin(w[p + "k"], h), H), heads(lin(w[p + "v"], h), H),
                          heads(dec, H))
    o = (rms_unit(o, eps) * w[p + "norm"]).reshape(h.shape[0], -1)
    return lin(w[p + "o"], o * silu(lin(w[p + "g"], h)))


def right_lightning(w, p, m, h, eps):
    H = int(m["heads"])
    o = lightning_core(heads(silu(lin(w[p + "q"], h)), H), heads(silu(lin(w[p + "k"], h)), H),
                       heads(silu(lin(w[p + "v"], h)), H), torch.tensor(m["decay"], dtype=F64))
    o = rms_unit(o.reshape(h.shape[0], -1), eps) * w[p + "norm"]
    return lin(w[p + "o"], o * torch.sigmoid(lin(w[p + "g"], h)))


def mixer(w, p, entry, h, eps):
    m = entry["mixer"]
    if entry["type"] == "parallel":
        a, b = left_talk(w, p + "left.", m["left"], h), right_gated(w, p + "right.", m["right"], h, eps)
    else:
        a, b = left_softmax(w, p + "left.", m["left"], h), right_lightning(w, p + "right.", m["right"], h, eps)
    return 0.5 * (rms_unit(a, eps) * w[p + "left.out"] + rms_unit(b, eps) * w[p + "right.out"])


def dense(w, p, h):
    return lin(w[p + "down"], silu(lin(w[p + "gate"], h)) * lin(w[p + "up"], h))


# ------------------------------------------------------------------ model
def forward(cfg: dict, w: dict, tokens, layers: bool = False):
    """Logits [T, V] of every position (float64); with ``layers`` also the stream after every layer."""
    eps = float(cfg["norm"]["eps"])
    x = embed(w, tokens, float(cfg["embedding"]["scale"]))
    streams = []
    for i, e in enumerate(cfg["layers"]):
        p = f"l{i}."
        x = x + mixer(w, p + "mix.", e, rms_unit(x, eps) * w[p + "norm1"], eps)
        if e.get("mlp") is not None:
            x = x + dense(w, p + "mlp.", rms_unit(x, eps) * w[p + "norm2"])
        streams.append(x.clone())
    y = lin(w["embed"], rms_unit(x, eps) * w["final.norm"])
    return (y, streams) if layers else y
