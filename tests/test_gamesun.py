"""Gamesun in the framework against the plain float64 oracle (tests/gamesun_oracle.py): every mechanism
alone, then the model through the engine's scheduler, block pool, state slots and step — whole prompts,
token-by-token decoding, portions down to two tokens, unequal batches, reused pages and slots, keys at
window and page borders, far memories, first tokens, long decoding, other geometries, greedy generation,
the checkpoint layout and the trace runner.  The same tests run the CPU reference ops here and the HIP
kernels on a GPU box."""
import copy
import json
import os
import subprocess
import sys

import pytest
import torch

import gamesun_oracle as orc
from dgi.engine import EngineConfig, LLMEngine
from dgi.models.config import (AttentionSpec, GamesunConfig, GatedLinearSpec, GluSpec, LayerSpec, LightningSpec, ParallelSpec,
                               get_config)
from dgi.ops import linrec, mix
from dgi.sched.request import SamplingParams

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
DEVICES = ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)]
F64 = torch.float64
I32 = torch.int32


# ----------------------------------------------------------------------------------- helpers
def attn(heads, kv, dim, vdim, scale, window, talk):
    return AttentionSpec(heads, kv, dim, vdim, scale, None, "window" if window else "causal", window, out_gate=False,
                         qk_norm="none", qk_norm_weight=False, weights="sigmoid" if talk else "softmax", talk=talk,
                         head_temp=not talk, bias=talk)


def glayer(heads, kv, dim, vdim, scale, window, right, ff):
    """Talking-heads sigmoid attention beside gated linear attention ``right`` = (heads, dim, vdim, tau, rank)."""
    return LayerSpec("parallel", ParallelSpec(attn(heads, kv, dim, vdim, scale, window, True), GatedLinearSpec(*right)),
                     GluSpec(ff, act="silu") if ff else None)


def llayer(heads, kv, dim, vdim, scale, window, right, ff):
    """Softmax attention with temperatures beside lightning attention ``right`` = (heads, dim, vdim, decays)."""
    return LayerSpec("parallel_2", ParallelSpec(attn(heads, kv, dim, vdim, scale, window, False), LightningSpec(*right)),
                     GluSpec(ff, act="silu") if ff else None)


def small_cfg(**kw) -> GamesunConfig:
    """Four layers that differ in everything: windows, scales, heads (== kv heads, three query heads per kv head), key
    size != value size, recurrences with other head counts than their attention, a layer without feed-forward."""
    args = dict(name="t", vocab_size=59, hidden_size=32, layers=[
        glayer(6, 2, 8, 12, 0.4, 9, (2, 10, 6, 3.0, 5), 20),
        llayer(2, 2, 12, 8, 0.3, 21, (3, 4, 20, [0.5, 0.9, 0.999]), 0),
        llayer(4, 1, 8, 16, 0.5, 5, (1, 16, 12, [0.97]), 28),
        glayer(3, 3, 16, 8, 0.2, 30, (4, 6, 10, 16.0, 3), 12),
    ], embedding_scale=5.0, norm_eps=1e-5, max_position=64)
    args.update(kw)
    return GamesunConfig(**args)


def engine(cfg, device, dtype=torch.float32, num_blocks=96, bs=4, seed=3, max_len=256, seqs=4, graphs=False):
    return LLMEngine(EngineConfig(model="gamesun-test", device=device, dtype=dtype, block_size=bs, num_blocks=num_blocks,
                                  max_num_seqs=seqs, max_model_len=max_len, max_num_batched_tokens=max_len,
                                  enable_prefix_caching=True, use_graphs=graphs, token_align=0, decode_lookahead=graphs,
                                  seed=seed, graph_buckets=(1, 2, 4) if graphs else None), model_cfg=copy.deepcopy(cfg))


def toks(n, seed=0, vocab=59):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, vocab, (n,), generator=g).tolist()


def config_dict(cfg: GamesunConfig) -> dict:
    """The design's config.json for ``cfg``."""
    layers = []
    for l in cfg.layers:
        a, r = l.mixer.left, l.mixer.right
        lf = {"heads": a.heads, "kv_heads": a.kv_heads, "dim": a.dim, "vdim": a.vdim, "scale": a.scale}
        if a.window:
            lf["mask"] = {"size": a.window}
        rt = {"heads": r.heads, "dim": r.dim, "vdim": r.vdim}
        rt.update({"tau": r.tau} if l.type == "parallel" else {"decay": list(r.decay)})
        layers.append({"type": l.type, "mixer": {"left": lf, "right": rt},
                       "mlp": None if l.mlp is None else {"kind": "dense", "ff": l.mlp.ff}})
    return {"architecture": "Gamesun", "vocab": cfg.vocab_size, "width": cfg.hidden_size, "norm": {"eps": cfg.norm_eps},
            "embedding": {"scale": cfg.embedding_scale}, "layers": layers}


def params(model) -> dict:
    """The model's weights under the checkpoint's tensor names (CPU, model dtype)."""
    P = {"embed": model.embed, "final.norm": model.final_norm}
    for i, L in enumerate(model.layers):
        p, lf, rt = f"l{i}.", f"l{i}.mix.left.", f"l{i}.mix.right."
        a, r, f = L.spec.mixer.left, L.spec.mixer.right, L.spec.mlp
        c = 0
        for key, rows in ((lf + "q", a.q_size), (lf + "k", a.k_size), (lf + "v", a.v_size), (rt + "q", r.qk_size),
                          (rt + "k", r.qk_size), (rt + "v", r.inner), (rt + "g", r.inner)):
            P[key] = L.in_proj[c:c + rows]
            if L.in_bias is not None and key.startswith(lf):
                P[key + ".b"] = L.in_bias[c:c + rows]
            c += rows
        P[p + "norm1"] = L.norm1
        for key, t in ((lf + "o", L.o_left), (lf + "o.b", L.o_bias), (lf + "talk", L.talk), (lf + "pb", L.pb), (lf + "temp", L.temp),
                       (lf + "out", L.out_left), (rt + "o", L.o_right), (rt + "norm", L.rnorm), (rt + "out", L.out_right),
                       (rt + "a1", L.a1), (rt + "a2", L.a2), (rt + "a2.b", L.a2_b)):
            if t is not None:
                P[key] = t
        if f is not None:
            P[p + "norm2"] = L.norm2
            P[p + "mlp.gate"], P[p + "mlp.up"], P[p + "mlp.down"] = L.gate_up[:f.ff], L.gate_up[f.ff:], L.down
    return {k: v.detach().cpu().contiguous() for k, v in P.items()}


def oracle_logits(eng, tokens, layers=False):
    P = {k: v.to(F64) for k, v in params(eng.model).items()}
    return orc.forward(config_dict(eng.model_cfg), P, tokens, layers)


def feed_all(eng, rid, tokens, cuts):
    """Feed `tokens` in portions of the given sizes (the rest one by one); logits of every position."""
    out, at = [], 0
    for n in list(cuts) + [1] * len(tokens):
        if at >= len(tokens):
            break
        part = tokens[at:at + n]
        out.append(eng.feed([(rid, part, list(range(len(part))))])[0])
        at += len(part)
    return torch.cat(out, 0)


def close(a, b, tol):
    assert a.shape == b.shape
    err = (a.double().cpu() - b.double().cpu()).abs().max().item()
    assert err <= tol, f"max abs difference {err} > {tol}"


def seq_meta(lens, starts, slots, device):
    pos, r0 = [], [0]
    for n, s in zip(lens, starts):
        pos += list(range(s, s + n))
        r0.append(r0[-1] + n)
    mk = lambda x: torch.tensor(x, dtype=I32, device=device)   # noqa: E731
    return mk(pos), mk(r0), mk(slots)


def portions(n, cuts, other_n):
    """(rows of sequence a, rows of sequence b) per step: a in the given cuts then whole, b five rows now and then."""
    at_a = at_b = 0
    for i, c in enumerate(list(cuts) + [n]):
        na = min(c, n - at_a)
        nb = min(5, other_n - at_b) if i % 2 else 0
        if na or nb:
            yield at_a, na, at_b, nb
        at_a, at_b = at_a + na, at_b + nb


def paged(ks, vs, bs, dtype, device, g):
    """Shuffled pages filled with the given keys / values (lists of [n, G, d]); unused entries hold large garbage."""
    pages = [-(-k.shape[0] // bs) for k in ks]
    nb = sum(pages) + 3
    perm = (torch.randperm(nb - 1, generator=g) + 1).tolist()
    G, dk, dv = ks[0].shape[1], ks[0].shape[2], vs[0].shape[2]
    kc = torch.full((nb, G, bs, dk), 900.0, dtype=dtype)
    vc = torch.full((nb, G, bs, dv), 900.0, dtype=dtype)
    bt = torch.zeros(len(ks), max(pages), dtype=I32)
    for i, (k, v) in enumerate(zip(ks, vs)):
        for b in range(pages[i]):
            bt[i, b] = perm.pop()
        for j in range(k.shape[0]):
            kc[bt[i, j // bs], :, j % bs], vc[bt[i, j // bs], :, j % bs] = k[j], v[j]
    return bt.to(device), kc.to(device), vc.to(device)


# ----------------------------------------------------------------------------------- mechanisms
def test_configuration_from_the_file_form():
    cfg = small_cfg()
    back = GamesunConfig.from_dict(config_dict(cfg))
    for a, b in zip(back.layers, cfg.layers):
        assert a.type == b.type and a.mixer.left == b.mixer.left and a.mlp == b.mlp
    assert back.kv_layer_shapes() == [(2, 8, 12), (2, 12, 8), (1, 8, 16), (3, 16, 8)]
    assert back.layers[1].mlp is None and back.layers[2].mixer.right.decay == [0.97]
    assert back.layers[0].mixer.right.decay_rank == 0          # only the checkpoint's shapes give it
    assert back.embedding_scale == 5.0 and back.norm_eps == 1e-5
    for path, value in ((("type",), "attention"), (("mixer", "left", "kv_heads"), 4), (("mlp", "kind"), "moe")):
        d = config_dict(cfg)
        e = d["layers"][0]
        for k in path[:-1]:
            e = e[k]
        e[path[-1]] = value
        with pytest.raises(ValueError):
            GamesunConfig.from_dict(d)
    d = config_dict(cfg)
    d["layers"][1]["mixer"]["right"]["decay"] = [0.5]
    with pytest.raises(ValueError):
        GamesunConfig.from_dict(d)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("W", [1, 7, 32, 300])
def test_embedding_with_position_vector(device, dtype, W):
    g = torch.Generator().manual_seed(1)
    table = torch.randn(11, W, generator=g).to(dtype)
    pos = [0, 1, 2, 17, 4095, 70000, 1000003]
    ids = [3, 0, 10, 3, 5, 5, 1]
    want = torch.stack([table[i].to(F64) * 2.5 + orc.position_vector(p, W) for i, p in zip(ids, pos)], 0)
    got = mix.embed_sinusoid(torch.tensor(ids, device=device), torch.tensor(pos, dtype=I32, device=device), table.to(device), 2.5,
                             mix.sinusoid_freqs(W, device=device))
    close(got, want, 2e-6)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("G,dk,dv,lead", [(2, 8, 16, 8), (3, 5, 7, 3), (1, 64, 128, 0)])
def test_page_write(device, dtype, G, dk, dv, lead):
    """k | v columns of wider rows land at their slots; a row without a slot and all other entries stay as they were."""
    g = torch.Generator().manual_seed(2)
    T, bs, nb = 7, 4, 5
    u = torch.randn(T, lead + G * (dk + dv) + 8, generator=g).to(dtype)
    slots = torch.tensor([5, 19, 4, -1, 7, 12, 8], dtype=I32)
    kc, vc = torch.randn(nb, G, bs, dk, generator=g).to(dtype), torch.randn(nb, G, bs, dv, generator=g).to(dtype)
    wk, wv = kc.clone(), vc.clone()
    for t, s in enumerate(slots.tolist()):
        if s >= 0:
            wk[s // bs, :, s % bs] = u[t, lead:lead + G * dk].view(G, dk)
            wv[s // bs, :, s % bs] = u[t, lead + G * dk:lead + G * (dk + dv)].view(G, dv)
    kd, vd = kc.to(device), vc.to(device)
    mix.kv_rows(u.to(device)[:, lead:], slots.to(device), G, dk, dv, kd, vd)
    assert torch.equal(kd.cpu(), wk) and torch.equal(vd.cpu(), wv)


def edge_case(H, G, dk, dv, n, window, dtype, g, edge_rows, lo=0.2):
    """Queries that single out one key each, placed just inside and just outside their window (and far, and at page
    borders); its value is large, so seeing or missing it moves the output far beyond any tolerance."""
    q, k = torch.randn(n, H, dk, generator=g) * lo, torch.randn(n, G, dk, generator=g) * lo
    v = torch.randn(n, G, dv, generator=g) * 0.3
    for i, p in enumerate(edge_rows):
        for j in {max(0, p - window + 1), max(0, p - window)} if window else {0, p // 2}:
            u = torch.randn(dk, generator=g).sign()
            k[j] = u
            v[j] = 3.0 + i % 3
            q[p] = u * (1.0 + 0.1 * torch.arange(H)[:, None] / H)
    return q.to(dtype), k.to(dtype), v.to(dtype)


SIG_GEOMS = [(4, 2, 16, 32, 9), (6, 3, 24, 40, 64), (3, 1, 7, 5, 3), (9, 3, 16, 16, 1), (1, 1, 8, 16, 70), (16, 8, 64, 64, 33),
             (2, 2, 12, 8, 0), (20, 4, 32, 48, 17), (5, 5, 40, 24, 65)]


def talk_params(H, g):
    return torch.eye(H) * 0.9 + torch.randn(H, H, generator=g) * (0.4 / H ** 0.5), torch.linspace(-5.0, -1.0, H)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("geom", SIG_GEOMS, ids=lambda x: "-".join(map(str, x)))
def test_sigmoid_attention_rows(device, dtype, geom):
    """Mixed-head sigmoid attention over scattered pages: decode rows (keys in one run and cut into several) and a portion
    on cached keys, with one key per query at the window's edge that must be seen (or not)."""
    H, G, dk, dv, win = geom
    g = torch.Generator().manual_seed(3)
    n, bs = 150, 4
    rows = [149, 148, 130, 71, 70, 65, 64, 63, 33, 10, 9, 8, 2, 1, 0]
    q, k, v = edge_case(H, G, dk, dv, n, win, dtype, g, rows[:9])
    talk, pb = talk_params(H, g)
    scale = 8.0 / dk
    want = orc.talk_sigmoid_attention(q.to(F64), k.to(F64), v.to(F64), scale, talk.to(F64), pb.to(F64), win)
    if win:                                            # the case can tell a window that is one key off
        off = orc.talk_sigmoid_attention(q.to(F64), k.to(F64), v.to(F64), scale, talk.to(F64), pb.to(F64), win + 1)
        assert (off - want)[rows[:9]].abs().amax() > 0.5
    bt, kc, vc = paged([k], [v], bs, dtype, device, g)
    tol = (2e-5 if dtype == torch.float32 else 0.01) * max(1.0, want.abs().max().item())
    td, pd = talk.to(device), pb.to(device)
    qd = q.reshape(n, -1).to(device)
    pos = torch.tensor(rows, dtype=I32, device=device)
    for max_keys in (0, n):
        got = mix.sigmoid_attn_rows(qd[rows], kc, vc, bt.repeat(len(rows), 1), None, pos, H, G, scale, win, td, pd, max_keys=max_keys)
        close(got, want[rows].reshape(len(rows), -1), tol)
    p0 = 101
    got = mix.sigmoid_attn_rows(qd[p0:], kc, vc, bt, torch.tensor([0, n - p0], dtype=I32, device=device),
                                torch.arange(p0, n, dtype=I32, device=device), H, G, scale, win, td, pd)
    close(got, want[p0:].reshape(n - p0, -1), tol)
    plain = orc.talk_sigmoid_attention(q.to(F64), k.to(F64), v.to(F64), scale, torch.eye(H, dtype=F64), torch.zeros(H, dtype=F64), win)
    got = mix.sigmoid_attn_rows(qd[rows], kc, vc, bt.repeat(len(rows), 1), None, pos, H, G, scale, win)
    close(got, plain[rows].reshape(len(rows), -1), tol * max(1.0, plain.abs().max().item()))


MFMA_GEOMS = [(4, 2, 64, 128, 40), (4, 4, 32, 16, 0), (6, 2, 24, 48, 17), (8, 8, 128, 64, 100), (16, 8, 128, 128, 90),
              (12, 12, 40, 32, 33), (16, 2, 64, 96, 1), (32, 8, 64, 128, 50), (32, 8, 128, 128, 64), (24, 6, 96, 80, 31), (24, 8, 64, 64, 20),
              (1, 1, 8, 16, 5), (32, 16, 64, 64, 45)]


@pytest.mark.gpu
@pytest.mark.parametrize("geom", MFMA_GEOMS, ids=lambda x: "-".join(map(str, x)))
def test_mfma_sigmoid_prompt_attention(geom):
    """The MFMA prompt kernel: three portions in one step (on top of cached keys ending inside a key tile, a fresh one with
    rows past a 128-row tile, one of two rows), window edges singled out as above."""
    H, G, dk, dv, win = geom
    dev, bs, dtype = "cuda", 16, torch.bfloat16
    g = torch.Generator().manual_seed(4)
    lens, cached = [200, 150, 61], [101, 0, 59]
    talk, pb = talk_params(H, g)
    scale = 8.0 / dk
    qs, ks, vs, wants = [], [], [], []
    for n, c in zip(lens, cached):
        q, k, v = edge_case(H, G, dk, dv, n, win, dtype, g, [n - 1, n - 2, n - 20, c + 1])
        w = orc.talk_sigmoid_attention(q.to(F64), k.to(F64), v.to(F64), scale, talk.to(F64), pb.to(F64), win)
        wants.append(w[c:].reshape(n - c, -1))
        qs.append(q[c:].reshape(n - c, -1)), ks.append(k), vs.append(v)
    bt, kc, vc = paged(ks, vs, bs, dtype, dev, g)
    cu = torch.tensor([0, 99, 249, 251], dtype=I32, device=dev)
    u = torch.cat([torch.cat(qs, 0), torch.zeros(251, 8, dtype=dtype)], 1).to(dev)           # q columns of wider rows
    assert mix.sigmoid_prefill_ok(u, kc, vc, H, G)
    want = torch.cat(wants, 0)
    got = mix.sigmoid_prefill(u, kc, vc, bt, cu, torch.tensor(lens, dtype=I32, device=dev), H, G, scale, win, talk.to(dev), pb.to(dev))
    close(got, want, 0.012 * max(1.0, want.abs().max().item()))


def test_mfma_prompt_kernel_refuses_what_it_does_not_serve():
    q = torch.zeros(4, 64)
    assert not mix.sigmoid_prefill_ok(q, torch.zeros(2, 1, 16, 8), torch.zeros(2, 1, 16, 16), 1, 1)      # CPU tensors


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("geom", [(4, 2, 16, 32, 9), (3, 1, 7, 5, 3), (9, 1, 16, 16, 64), (2, 2, 64, 24, 0), (4, 2, 64, 64, 1)],
                         ids=lambda x: "-".join(map(str, x)))
def test_window_softmax_with_head_factors(device, dtype, geom):
    """Sliding window and a factor per head — above and below one, negative, zero — in the row kernels."""
    H, G, dk, dv, win = geom
    g = torch.Generator().manual_seed(5)
    n, bs = 140, 4
    rows = [139, 138, 100, 70, 64, 63, 17, 9, 8, 1, 0]
    q, k, v = edge_case(H, G, dk, dv, n, win, dtype, g, rows[:7])
    temp = torch.tensor([1.7, -0.6, 0.0, 0.4, 2.0, 1.0, -1.5, 0.2, 3.0])[:H]
    scale = 6.0 / dk
    want = orc.temp_softmax_attention(q.to(F64), k.to(F64), v.to(F64), scale, temp.to(F64), win)
    bt, kc, vc = paged([k], [v], bs, dtype, device, g)
    tol = (2e-5 if dtype == torch.float32 else 0.01) * max(1.0, want.abs().max().item())
    pos = torch.tensor(rows, dtype=I32, device=device)
    qd = q.reshape(n, -1).to(device)
    got = mix.masked_attn_rows(qd[rows], kc, vc, bt.repeat(len(rows), 1), None, pos, H, G, scale, 0, None, window=win,
                               head_scale=temp.to(device))
    close(got, want[rows].reshape(len(rows), -1), tol)
    p0 = 77
    got = mix.masked_attn_rows(qd[p0:], kc, vc, bt, torch.tensor([0, n - p0], dtype=I32, device=device),
                               torch.arange(p0, n, dtype=I32, device=device), H, G, scale, 0, None, window=win,
                               head_scale=temp.to(device))
    close(got, want[p0:].reshape(n - p0, -1), tol)


@pytest.mark.gpu
@pytest.mark.parametrize("hd,hv,win", [(64, 64, 30), (128, 128, 70), (64, 64, 1), (128, 128, 0), (64, 128, 40), (128, 64, 33),
                                       (48, 96, 70), (40, 24, 17), (96, 72, 100), (8, 8, 5), (72, 128, 0), (16, 40, 64)])
@pytest.mark.parametrize("bs", [16, 32])
def test_mfma_window_softmax_with_head_factors(hd, hv, win, bs):
    H, G, dev, dtype = 4, 2, "cuda", torch.bfloat16
    g = torch.Generator().manual_seed(6)
    lens, cached = [200, 150], [101, 0]
    temp = torch.tensor([1.7, -0.6, 0.0, 0.4])
    scale = 6.0 / hd
    qs, ks, vs, wants = [], [], [], []
    for n, c in zip(lens, cached):
        q, k, v = edge_case(H, G, hd, hv, n, win, dtype, g, [n - 1, n - 2, n - 20, c + 1])
        w = orc.temp_softmax_attention(q.to(F64), k.to(F64), v.to(F64), scale, temp.to(F64), win)
        wants.append(w[c:].reshape(n - c, -1))
        qs.append(q[c:].reshape(n - c, -1)), ks.append(k), vs.append(v)
    bt, kc, vc = paged(ks, vs, bs, dtype, dev, g)
    cu = torch.tensor([0, 99, 249], dtype=I32, device=dev)
    want = torch.cat(wants, 0)
    got = mix.paged_prefill_masked(torch.cat(qs, 0).to(dev), kc, vc, bt, cu, torch.tensor(lens, dtype=I32, device=dev), H, G,
                                   scale, 0, None, window=win, head_scale=temp.to(dev))
    close(got, want, 0.012 * max(1.0, want.abs().max().item()))


SCAN_GEOMS = [(2, 12, 12), (3, 64, 64), (1, 5, 7), (2, 130, 30), (4, 6, 10), (2, 48, 70), (1, 300, 17), (2, 16, 130), (1, 1, 1)]


def scan_case(mode, H, D, V, n, dtype, g):
    """(q, k, v, decays, oracle output); gla: a decay per token and channel, light: one per head."""
    q, k, v = (torch.randn(n, H * d, generator=g).to(dtype) for d in (D, D, V))
    q64, k64, v64 = (x.to(F64).view(n, H, -1) for x in (q, k, v))
    if mode == "gla":
        dec = torch.rand(n, H * D, generator=g) ** 0.1
        return q, k, v, dec, orc.gated_linear_core(q64 * D ** -0.5, k64, v64, dec.to(F64).view(n, H, D)).reshape(n, -1)
    dec = torch.rand(H, generator=g) ** 0.1
    return q, k, v, dec, orc.lightning_core(orc.silu(q64), orc.silu(k64), orc.silu(v64), dec.to(F64)).reshape(n, -1)


def scan_call(mode, qkv, dec, S, meta, H, D, V):
    q, k, v = qkv[:, :H * D], qkv[:, H * D:2 * H * D], qkv[:, 2 * H * D:]
    return (linrec.gla_scan if mode == "gla" else linrec.lightning_scan)(q, k, v, dec, S, *meta, H, D, V)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("mode", ["gla", "light"])
@pytest.mark.parametrize("geom", SCAN_GEOMS, ids=lambda x: "-".join(map(str, x)))
def test_recurrences_portions_and_slots(device, dtype, mode, geom):
    """Whole sequence == portions of 1, 2, 7, ... rows through a slot that held another state before, with a second
    sequence in the same step; q | k | v are row views of one wider buffer."""
    H, D, V = geom
    g = torch.Generator().manual_seed(7)
    n = 37
    qa, ka, va, da, want_a = scan_case(mode, H, D, V, n, dtype, g)
    qb, kb, vb, db, _w = scan_case(mode, H, D, V, n, dtype, g)
    if mode == "light":
        db = da
    x = [t.to(F64).view(n, H, -1) for t in (qb, kb, vb)]
    want_b = (orc.gated_linear_core(x[0] * D ** -0.5, x[1], x[2], db.to(F64).view(n, H, D)) if mode == "gla" else
              orc.lightning_core(*(orc.silu(t) for t in x), db.to(F64))).reshape(n, -1)
    S = (torch.randn(6, H, D, V, generator=g) * 50).to(device)
    got_a, got_b = [], []
    for at_a, na, at_b, nb in portions(n, [1, 1, 2, 7, 1, 9, 3], n):
        lens, starts, slots, rows, decs = [], [], [], [], []
        for cnt, at, slot, src, d in ((na, at_a, 3, (qa, ka, va), da), (nb, at_b, 5, (qb, kb, vb), db)):
            if cnt:
                lens.append(cnt), starts.append(at), slots.append(slot)
                rows.append(torch.cat([t[at:at + cnt] for t in src], 1))
                decs.append(d[at:at + cnt] if mode == "gla" else d)
        meta = seq_meta(lens, starts, slots, device)
        dec = (torch.cat(decs, 0) if mode == "gla" else da).to(device)
        y = scan_call(mode, torch.cat(rows, 0).to(device), dec, S, meta, H, D, V)
        got_a.append(y[:na])
        got_b.append(y[na:])
    for got, want in ((torch.cat(got_a, 0), want_a), (torch.cat(got_b, 0), want_b)):
        close(got, want[:got.shape[0]], 3e-5 * max(1.0, want.abs().max().item()))


@pytest.mark.gpu
@pytest.mark.parametrize("mode", ["gla", "light"])
@pytest.mark.parametrize("heads,n", [(6, 9), (48, 9), (64, 9), (4, 150), (32, 70)])
def test_recurrences_prompt_steps_of_every_grid_size(mode, heads, n):
    """A prompt step picks its layout by the number of workgroups and its length; five sequences continue a state."""
    H, D, V, ns = heads, 64, 64, 5
    g = torch.Generator().manual_seed(heads)
    S0 = torch.randn(ns + 1, H, D, V, generator=g) * 0.3
    cases = [scan_case(mode, H, D, V, n, torch.float32, g) for _ in range(ns)]
    qkv = torch.cat([torch.cat(c[:3], 1) for c in cases], 0)
    dec = torch.cat([c[3] for c in cases], 0) if mode == "gla" else cases[0][3]
    out = []
    for device in ("cpu", "cuda"):
        S = S0.clone().to(device)
        y = scan_call(mode, qkv.to(device), dec.to(device), S, seq_meta([n] * ns, [3] * ns, list(range(1, ns + 1)), device), H, D, V)
        out.append((y.cpu(), S.cpu()))
    for a, b in zip(*out):
        close(a, b, 3e-5 * max(1.0, b.abs().max().item()))


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("mode", ["gla", "light"])
@pytest.mark.parametrize("geom", [(2, 64, 32), (1, 130, 20), (3, 20, 16)], ids=lambda x: "-".join(map(str, x)))
def test_recurrences_with_decays_beyond_the_fp32_range(device, mode, geom):
    """Decays down to zero and to 1e-30, whose products over a few tokens leave the fp32 range, beside channels that
    barely decay: portions long enough for the chunked form, short ones and single tokens agree with the oracle."""
    H, D, V = geom
    g = torch.Generator().manual_seed(14)
    n = 150
    q, k, v = (torch.randn(n, H * d, generator=g) for d in (D, D, V))
    x = [t.to(F64).view(n, H, -1) for t in (q, k, v)]
    if mode == "gla":
        dec = torch.rand(n, H * D, generator=g) ** 0.05
        dec[20:40, ::3] = 1e-3                         # a few tokens of strong decay, then none
        dec[45, 1::2] = 1e-30
        dec[50:53, 0] = 0.0
        dec[70:, :5] = 0.9999
        dec[100:, 7] = 0.02
        want = orc.gated_linear_core(x[0] * D ** -0.5, x[1], x[2], dec.to(F64).view(n, H, D)).reshape(n, -1)
    else:
        dec = torch.tensor([0.01, 0.0, 0.999])[:H]
        want = orc.lightning_core(*(orc.silu(t) for t in x), dec.to(F64)).reshape(n, -1)
    S = torch.full((3, H, D, V), 77.0, device=device)
    out, at = [], 0
    for c in [37, 1, 64, 3, 2, 40, 3]:
        r = slice(at, at + c)
        out.append(scan_call(mode, torch.cat([q[r], k[r], v[r]], 1).to(device), (dec[r] if mode == "gla" else dec).to(device), S,
                             seq_meta([c], [at], [1], device), H, D, V))
        at += c
    assert at == n
    close(torch.cat(out, 0), want, 3e-5 * max(1.0, want.abs().max().item()))


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("mode", ["gla", "light"])
def test_recurrences_remember_a_far_token(device, mode):
    """One early token writes a large value under a key that only the last query asks for, hundreds of tokens later,
    through prompt portions and many decode steps: a lost or reset state shows at once."""
    H, D, V, n, far = 2, 8, 8, 400, 7
    g = torch.Generator().manual_seed(9)
    q, k, v = torch.full((n, H * D), -30.0), torch.full((n, H * D), -30.0), torch.randn(n, H * V, generator=g) * 0.1
    if mode == "gla":
        q.zero_(), k.zero_()
    k[:, 1::D] = 1.0                                  # every token writes under channel 1 of each head
    k[far, 1::D] = k[far, 2]
    k[far, 0::D] = 1.0                                # ... but the far token under channel 0
    v[far] = 9.0
    q[:, 1::D] = 1.0
    q[n - 1, 1::D] = q[n - 1, 2]
    q[n - 1, 0::D] = 1.0                              # only the last query reads channel 0
    q64, k64, v64 = (t.to(F64).view(n, H, -1) for t in (q, k, v))
    if mode == "gla":
        dec = torch.full((n, H * D), 0.9995)
        want = orc.gated_linear_core(q64 * D ** -0.5, k64, v64, dec.to(F64).view(n, H, D)).reshape(n, -1)
    else:
        dec = torch.tensor([0.9995, 0.999])
        want = orc.lightning_core(orc.silu(q64), orc.silu(k64), orc.silu(v64), dec.to(F64)).reshape(n, -1)
    assert want[n - 1].abs().min() > 0.5              # the far value is what the last query reads
    S = torch.zeros(3, H, D, V, device=device)
    out, at = [], 0
    for c in [50, 2, 200] + [1] * 148:
        r = slice(at, at + c)
        out.append(scan_call(mode, torch.cat([q[r], k[r], v[r]], 1).to(device), (dec[r] if mode == "gla" else dec).to(device), S,
                             seq_meta([c], [at], [2], device), H, D, V))
        at += c
    assert at == n
    close(torch.cat(out, 0), want, 1e-4 * max(1.0, want.abs().max().item()))


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("T,W,rank,N,tau", [(5, 32, 3, 20, 16.0), (1, 300, 17, 7, 1.0), (1100, 72, 16, 40, 3.0), (3, 40, 1, 300, 0.5),
                                             (33, 64, 20, 52, 2.0), (1030, 96, 4, 33, 16.0), (17, 32, 16, 300, 5.0)])
def test_lowrank_decay(device, dtype, T, W, rank, N, tau):
    g = torch.Generator().manual_seed(10)
    h = torch.randn(T, W, generator=g).to(dtype)
    a1, a2, b = torch.randn(rank, W, generator=g) * 0.3, torch.randn(N, rank, generator=g), torch.randn(N, generator=g) * 3
    b[0], b[-1] = 60.0, -60.0                          # far in both saturated ends
    want = orc.channel_decay(orc.lin(a2.to(F64), orc.lin(a1.to(F64), h.to(F64))) + b.to(F64), tau)
    close(linrec.lowrank_decay(h.to(device), a1.to(device), a2.to(device), b.to(device), tau), want, 1e-5)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("W", [32, 300, 1024, 2500, 4096])
def test_branch_norms_residual_and_next_norm(device, dtype, W):
    g = torch.Generator().manual_seed(11)
    if W == 2500 and device == "cuda":
        W = 2504                                       # beyond 2048 columns rows come in multiples of four
    x = torch.randn(5, W, generator=g) * 3
    a, b = (torch.randn(5, W, generator=g) * 4).to(dtype), torch.randn(5, W, generator=g).to(dtype)
    wa, wb, wn = (torch.randn(W, generator=g) for _ in range(3))
    want = x.to(F64) + 0.5 * (orc.rms_unit(a.to(F64), 1e-5) * wa.to(F64) + orc.rms_unit(b.to(F64), 1e-5) * wb.to(F64))
    for nxt in (wn, None):
        xd = x.clone().to(device)
        y = linrec.pair_add_norm(xd, a.to(device), b.to(device), wa.to(device), wb.to(device), None if nxt is None else nxt.to(device),
                                 1e-5, torch.float32)
        close(xd, want, 2e-5)
        close(y, want if nxt is None else orc.rms_unit(want, 1e-5) * nxt.to(F64), 4e-5)
    xd = x.clone().to(device)
    assert linrec.pair_add_norm(xd, a.to(device), b.to(device), wa.to(device), wb.to(device), None, 1e-5) is None
    close(xd, want, 2e-5)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("H,dv,gate", [(4, 24, "silu"), (1, 96, "sigmoid"), (1, 1024, "sigmoid"), (1, 2048, "sigmoid"), (1, 1500, "silu")])
def test_read_out_norm_over_a_head_and_over_all_heads(device, H, dv, gate):
    g = torch.Generator().manual_seed(12)
    y, w = torch.randn(9, H * dv, generator=g) * 2, torch.randn(dv, generator=g)
    z = torch.randn(9, H * dv + 8, generator=g).bfloat16()[:, 8:]
    u = (orc.rms_unit(y.to(F64).view(9, H, dv), 1e-5) * w.to(F64)).reshape(9, -1)
    zf = z.to(F64)
    want = u * (orc.silu(zf) if gate == "silu" else torch.sigmoid(zf))
    close(linrec.head_norm_gate(y.to(device), z.to(device), w.to(device), H, 1e-5, gate, torch.float32), want, 3e-5)


# ----------------------------------------------------------------------------------- the model
@pytest.mark.parametrize("device", DEVICES)
def test_layer_streams_match_oracle(device):
    eng = engine(small_cfg(), device)
    t = toks(43, 1)
    n = len(eng.model_cfg.layers)
    eng.model.capture_layers = tuple(range(n))
    got = eng.feed([("a", t, list(range(len(t))))], ["a"])[0]
    eng.model.capture_layers = ()
    want, streams = oracle_logits(eng, t, True)
    for r in range(n):
        close(eng.model.captured[r], streams[r], 1e-4 * max(1.0, streams[r].abs().max().item()))
    close(got, want, 3e-4)


BASE = small_cfg().layers
VARIANTS = {
    "base": {},
    "reversed": {"layers": BASE[::-1], "embedding_scale": 1.0, "norm_eps": 1e-2},
    "gated_only": {"layers": [BASE[0], BASE[3]]},
    "lightning_only": {"layers": [BASE[1], BASE[2]]},
    "windows_of_one": {"layers": [glayer(2, 1, 8, 8, 0.5, 1, (2, 4, 4, 2.0, 2), 8), llayer(2, 1, 8, 8, 0.5, 1, (2, 4, 4, [0.9, 0.99]), 8)]},
    "no_window": {"layers": [glayer(2, 1, 8, 8, 0.5, 0, (2, 4, 4, 2.0, 2), 8), llayer(2, 1, 8, 8, 0.5, 0, (2, 4, 4, [0.9, 0.99]), 8)]},
    "ones": {"layers": [glayer(1, 1, 1, 1, 1.0, 3, (1, 1, 1, 1.0, 1), 1), llayer(1, 1, 1, 1, 1.0, 2, (1, 1, 1, [0.5]), 0)],
             "hidden_size": 6},
    "odd_width": {"layers": [glayer(3, 1, 5, 7, 0.4, 6, (2, 3, 9, 4.0, 2), 11), llayer(2, 2, 3, 5, 0.6, 7, (3, 7, 3, [0.3, 0.8, 1.0]), 9)],
                  "hidden_size": 27},
}


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("variant", list(VARIANTS))
def test_whole_decode_and_portions_match_oracle(device, variant):
    """Whole prompt, token by token, and portions of several sizes (down to two tokens, across pages and windows): all
    equal the oracle; other layer orders, constants, windows and sizes of one too."""
    eng = engine(small_cfg(**VARIANTS[variant]), device)
    t = toks(45, 2)
    want = oracle_logits(eng, t)
    tol = 3e-4 * max(1.0, want.abs().max().item() / 4)
    close(eng.feed([("w", t, list(range(len(t))))], ["w"])[0], want, tol)
    for name, cuts in (("d", [1]), ("p", [2, 2, 7, 3, 16, 2, 5]), ("q", [30, 2]), ("r", [1, 13])):
        got = feed_all(eng, name, t, cuts)
        eng.feed([], [name])
        close(got, want, tol)
    assert eng.pool.num_used == 0 and eng.state_pool.num_free == 4


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_unequal_batches_reuse_pages_and_slots(device, dtype):
    """Six requests of different lengths through four slots and a pool too small for all of them: portions beside single
    tokens, requests sitting steps out, pages and slots used again — every position equals the request run alone."""
    eng = engine(small_cfg(), device, dtype=dtype, num_blocks=40, bs=4)
    solo = engine(small_cfg(), device, dtype=dtype)
    solo.model.copy_from(eng.model)
    lens = {"a": 41, "b": 7, "c": 30, "d": 2, "e": 23, "f": 35}
    seqs = {k: toks(n, 10 + i) for i, (k, n) in enumerate(lens.items())}
    want = {k: solo.feed([(k, v, list(range(len(v))))], [k])[0] for k, v in seqs.items()}
    plan = [[("a", 5), ("b", 2)], [("a", 1), ("b", 1), ("c", 9), ("d", 2)], [("a", 17), ("c", 1)],
            [("b", 4), ("c", 2), ("a", 1), ("e", 3)], [("e", 20), ("a", 17)], [("c", 18), ("f", 6)],
            [("f", 1), ("c", 0)], [("f", 28)]]
    at = {k: 0 for k in seqs}
    got = {k: [] for k in seqs}
    for step in plan:
        entries, end = [], []
        for k, n in step:
            part = seqs[k][at[k]:at[k] + n]
            entries.append((k, part, list(range(len(part)))))
            at[k] += n
            if at[k] == len(seqs[k]):
                end.append(k)
        for k, out in zip([e[0] for e in entries], eng.feed(entries, end)):
            got[k].append(out)
    assert at == lens and eng.pool.num_used == 0 and eng.state_pool.num_free == 4
    assert eng.state_pool.stats["allocs"] == 6
    for k in seqs:
        close(torch.cat(got[k], 0), want[k], 2e-4 if dtype == torch.float32 else 0.08 * max(1.0, want[k].abs().max().item()))
    if dtype == torch.float32:
        close(want["a"], oracle_logits(solo, seqs["a"]), 3e-4)


@pytest.mark.parametrize("device", DEVICES)
def test_first_tokens_and_long_decoding(device):
    eng = engine(small_cfg(), device, max_len=256)
    t = toks(140, 5)
    want = oracle_logits(eng, t)
    close(eng.feed([("one", t[:1], [0])], ["one"])[0], want[:1], 2e-4)            # a sequence of one token
    close(eng.feed([("two", t[:2], [0, 1])], ["two"])[0], want[:2], 2e-4)
    got = feed_all(eng, "x", t, [3])                                              # 137 single-token steps, past every window
    close(got, want, 5e-4)


def sharp(model, layer=0, gain=6.0):
    """Make a layer's attention look for repeats: keys and queries from the same projection, so a token's score stands out
    at its own earlier occurrences; values grow, so that seeing or missing such a key moves the logits."""
    L = model.layers[layer]
    a = L.spec.mixer.left
    q = L.in_proj[: a.q_size].view(a.heads, a.dim, -1)
    k = L.in_proj[a.q_size: a.q_size + a.k_size].view(a.kv_heads, a.dim, -1)
    for h in range(a.heads):
        q[h] = k[h // (a.heads // a.kv_heads)] * gain
    L.in_proj[a.q_size + a.k_size: a.q_size + a.k_size + a.v_size] *= 3.0


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("kind", ["sigmoid", "softmax"])
def test_window_edges_through_the_model(device, kind):
    """A marked token placed just inside and just outside the windows of later queries, in prompt portions and decoded
    one by one; an oracle whose window is one off must disagree visibly."""
    win = 22
    layer = glayer(2, 1, 16, 8, 0.3, win, (1, 4, 4, 2.0, 2), 0) if kind == "sigmoid" else \
        llayer(2, 1, 16, 8, 0.3, win, (1, 4, 4, [0.9]), 0)
    eng = engine(small_cfg(layers=[layer]), device, max_len=160)
    sharp(eng.model)
    if kind == "sigmoid":
        eng.model.layers[0].pb.fill_(-5.0)
    t = [x % 50 for x in toks(130, 6)]
    for j, (far, mark) in enumerate(((win - 1, 55), (win, 56), (win - 1, 57), (win, 58))):
        p = 30 + 23 * j
        t[p], t[p + far] = mark, mark
    want = oracle_logits(eng, t)
    P = {k: v.to(F64) for k, v in params(eng.model).items()}
    for off in (win - 1, win + 1):
        cd = config_dict(eng.model_cfg)
        cd["layers"][0]["mixer"]["left"]["mask"]["size"] = off
        assert (orc.forward(cd, P, t) - want).abs().amax() > 0.05
    close(eng.feed([("w", t, list(range(len(t))))], ["w"])[0], want, 5e-4)
    close(feed_all(eng, "d", t, [29]), want, 5e-4)
    eng.feed([], ["d"])
    close(feed_all(eng, "p", t, [2, 7, 43, 2, 2, 31, 5]), want, 5e-4)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("kind", ["gla", "lightning"])
def test_far_memory_through_the_model(device, kind):
    """Only the recurrence reaches beyond a window of three: with slow decays, changing one early token moves the logits
    hundreds of positions later, and portions, decoding and the oracle agree on them."""
    layer = glayer(1, 1, 4, 4, 0.5, 3, (2, 8, 8, 400.0, 2), 0) if kind == "gla" else \
        llayer(1, 1, 4, 4, 0.5, 3, (2, 8, 8, [0.9995, 0.9999]), 0)
    eng = engine(small_cfg(layers=[layer]), device, max_len=400, num_blocks=120)
    t = toks(330, 8)
    other = list(t)
    other[4] = (t[4] + 1) % 59
    want = oracle_logits(eng, t)
    assert (oracle_logits(eng, other)[-1] - want[-1]).abs().amax() > 2e-3
    got = torch.cat([eng.feed([("a", t[:257], list(range(257)))])[0], feed_all(eng, "a", t[257:], [2, 40])], 0)
    close(got, want, 3e-4)


@pytest.mark.parametrize("device", DEVICES)
def test_greedy_generation_through_the_scheduler(device):
    eng = engine(small_cfg(), device, max_len=128)
    prompts = [toks(9, 20), toks(17, 21), toks(3, 22)]
    reqs = eng.generate(prompts, SamplingParams(max_tokens=12, temperature=0.0, ignore_eos=True))
    assert eng.scheduler.radix is None                   # state-carrying models never resume from shared pages
    P = {k: v.to(F64) for k, v in params(eng.model).items()}
    cd = config_dict(eng.model_cfg)
    for p, r in zip(prompts, reqs):
        seq = list(p)
        assert len(r.output) == 12
        for tok in r.output:
            lg = orc.forward(cd, P, seq)[-1]
            top2 = torch.topk(lg, 2).values
            assert tok == int(lg.argmax()) or (top2[0] - top2[1]) < 1e-3
            seq.append(tok)
    assert eng.pool.num_used == 0 and eng.state_pool.num_free == 4


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_graph_decode_equals_eager_decode(dtype):
    """Decode steps replayed as hipGraphs produce the tokens of the eager engine; replays follow each other with eager
    prompt steps between them."""
    cfg = small_cfg()
    eager, graph = (engine(cfg, "cuda", dtype=dtype, max_len=128, graphs=x) for x in (False, True))
    graph.model.copy_from(eager.model)
    prompts = [toks(9, 60), toks(17, 61), toks(3, 62)]
    sp = SamplingParams(max_tokens=14, temperature=0.0, ignore_eos=True)
    want = [r.output for r in eager.generate(prompts, sp)]
    for _ in range(3):                                       # later batches reuse slots and replay again
        assert [r.output for r in graph.generate(prompts, sp)] == want
    assert graph.runner.graphs is not None and graph.runner.graphs.captured
    assert graph.state_pool.num_free == 4 and graph.pool.num_used == 0


@pytest.mark.gpu
def test_mfma_prompt_paths_in_the_model(monkeypatch):
    """bf16 prompt portions take the MFMA kernels: same logits as the row kernels on the same engine (portions on top of
    cached tokens, two prompts in one step)."""
    cfg = small_cfg(hidden_size=64, layers=[
        glayer(4, 2, 48, 96, 0.12, 70, (2, 16, 16, 8.0, 4), 64), llayer(4, 2, 64, 64, 0.125, 50, (2, 16, 16, [0.9, 0.99]), 0),
        llayer(2, 1, 128, 128, 0.09, 130, (1, 8, 32, [0.95]), 64), glayer(16, 4, 16, 32, 0.25, 33, (2, 16, 16, 8.0, 4), 0)])
    a, b = toks(200, 70), toks(90, 71)

    def run():
        eng = engine(cfg, "cuda", dtype=torch.bfloat16, num_blocks=64, bs=16, max_len=512)
        out = [eng.feed([("a", a[:150], list(range(150)))]),
               eng.feed([("a", a[150:], list(range(50))), ("b", b, list(range(90)))], ["a", "b"])]
        return torch.cat([o for step in out for o in step], 0)

    assert mix.masked_prefill_available()
    fast = run()
    monkeypatch.setattr(mix, "MASKED_PREFILL", False)
    slow = run()
    close(fast, slow, 0.06 * max(1.0, slow.abs().max().item()))


def test_preempted_sequence_recomputes_its_state():
    """A pool too small for two growing sequences: one is preempted, gives its slot back, and is recomputed from
    position 0 — its tokens equal the undisturbed run."""
    cfg = small_cfg()
    big = engine(cfg, "cpu", max_len=128)
    ref = big.generate([toks(20, 30), toks(22, 31)], SamplingParams(max_tokens=20, temperature=0.0, ignore_eos=True))
    tight = engine(cfg, "cpu", num_blocks=18, bs=4, max_len=128)
    tight.model.copy_from(big.model)
    got = tight.generate([toks(20, 30), toks(22, 31)], SamplingParams(max_tokens=20, temperature=0.0, ignore_eos=True))
    assert tight.scheduler.num_preemptions > 0
    assert [r.output for r in got] == [r.output for r in ref]


def test_positions_beyond_any_table():
    """The design has no longest position: an engine longer than the configuration's default serves and matches."""
    eng = engine(small_cfg(layers=[BASE[2]], max_position=8), "cpu", max_len=200)
    t = toks(90, 33)
    close(eng.feed([("a", t, list(range(90)))], ["a"])[0], oracle_logits(eng, t), 3e-4)


def write_checkpoint(eng, path):
    from safetensors.torch import save_file
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(config_dict(eng.model_cfg), f)
    save_file({k: v.to(torch.bfloat16).contiguous() for k, v in params(eng.model).items()},
              os.path.join(path, "model.safetensors"))


def test_checkpoint_layout_and_trace_runner(tmp_path):
    """config.json + safetensors in the design's naming -> registry, loader, engine; the replay command writes the
    logits of the wanted places, step by step."""
    src = engine(small_cfg(), "cpu", dtype=torch.bfloat16)          # bf16 weights survive the file bit for bit
    for L in src.model.layers:                                      # ... also those the model keeps in fp32
        for k, t in L.named():
            if k != "decay":
                t.copy_(t.to(torch.bfloat16).to(t.dtype))
    ck = str(tmp_path / "model")
    write_checkpoint(src, ck)
    cfg = get_config(ck)
    assert isinstance(cfg, GamesunConfig) and cfg.num_layers == 4
    eng = LLMEngine(EngineConfig(model=ck, device="cpu", dtype=torch.float32, block_size=4, num_blocks=64, max_num_seqs=4,
                                 max_model_len=128, max_num_batched_tokens=128, use_graphs=False, token_align=0))
    assert [eng.model_cfg.layers[i].mixer.right.decay_rank for i in (0, 3)] == [5, 3]      # from the tensors' shapes
    t = toks(21, 40)
    want = oracle_logits(eng, t)
    close(eng.feed([("a", t, list(range(len(t))))], ["a"])[0], want, 3e-4)
    out = tmp_path / "out"
    steps = [{"step": 0, "entries": [{"id": "x", "tokens": t[:6], "want": [0, 5]}, {"id": "y", "tokens": t[:2], "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "x", "tokens": t[6:7], "want": [0]}], "end": ["y"]},
             {"step": 2, "entries": [{"id": "x", "tokens": t[7:], "want": [13]}], "end": ["x"]}]
    r = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", ck, "--dtype", "float32", "--out",
                        str(out), "--max-tokens", "64", "--device", "cpu"], input="\n".join(json.dumps(s) for s in steps) + "\n",
                       capture_output=True, text=True, timeout=300)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [l for l in r.stdout.splitlines() if l.startswith("done")] == ["done 0", "done 1", "done 2"]
    import numpy as np
    for step, rows in ((0, [0, 5]), (1, [6]), (2, [20])):
        got = torch.from_numpy(np.fromfile(str(out / f"{step}.f32"), dtype="<f4").reshape(len(rows), -1))
        close(got, want[rows], 3e-4)


def test_preset_and_registry():
    cfg = get_config("gamesun-tiny")
    assert isinstance(cfg, GamesunConfig) and [l.type for l in cfg.layers] == ["parallel", "parallel_2"] * 2
    assert len(get_config("gamesun-tiny@L2").layers) == 2
    eng = LLMEngine(EngineConfig(model="gamesun-tiny", device="cpu", dtype=torch.float32, num_blocks=32, max_num_seqs=2,
                                 max_model_len=128, use_graphs=False))
    assert type(eng.model).__name__ == "GamesunModel" and eng.state_pool is not None
    r = eng.generate([toks(5, 1, 512)], SamplingParams(max_tokens=4, temperature=0.0, ignore_eos=True))
    assert len(r[0].output) == 4


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_kernels_match_the_reference_ops_on_a_prompt_batch(dtype):
    """The HIP kernels against the CPU reference ops through the same engine code, over a batch of portions and decode
    rows."""
    cfg = small_cfg()
    cpu, gpu = engine(cfg, "cpu", dtype=dtype), engine(cfg, "cuda", dtype=dtype)
    cpu.model.copy_from(gpu.model)
    a, b = toks(50, 50), toks(33, 51)
    for eng in (cpu, gpu):
        eng.out = [eng.feed([("a", a[:40], list(range(40))), ("b", b[:2], [0, 1])]),
                   eng.feed([("a", a[40:41], [0]), ("b", b[2:], list(range(31)))]),
                   eng.feed([("a", a[41:], list(range(9)))], ["a", "b"])]
    x = torch.cat([u for o in cpu.out for u in o], 0)
    y = torch.cat([v for o in gpu.out for v in o], 0).cpu()
    close(y, x, 3e-4 if dtype == torch.float32 else 0.08 * max(1.0, x.abs().max().item()))
