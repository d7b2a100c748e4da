"""Plain float64 definition of the Zupilorn decoder, one function per mechanism, and makers of small random
checkpoints.  It recomputes whole sequences (no cache, no batching, keys and values expanded per head, the
recurrence walked token by token, every expert applied to its scaled input) and shares no code with the engine;
the engine's tests compare against it."""

from __future__ import annotations

import json
import math
from pathlib import Path

import torch

F64 = torch.float64


# --------------------------------------------------------------------------- mechanisms
def sigmoid(x):
    return 1.0 / (1.0 + torch.exp(-x))


def unit(x, eps):
    """x over its root mean square."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def zero_norm(x, eps, w):
    """An RMS norm whose stored weight is the distance of its gain from one."""
    return unit(x, eps) * (1.0 + w)


def rotate_half(x, pos, base, dims):
    """x [T, n]: channels (i, i + dims/2), i < dims/2, turn by pos * base^(-2i/dims); the rest pass."""
    out = x.clone()
    half = dims // 2
    for i in range(half):
        a = pos.to(F64) * base ** (-2.0 * i / dims)
        u, v = x[:, i], x[:, i + half]
        out[:, i] = u * torch.cos(a) - v * torch.sin(a)
        out[:, i + half] = v * torch.cos(a) + u * torch.sin(a)
    return out


def depth_average(streams, coef):
    """sum_j coef[j] * streams[j]"""
    total = torch.zeros_like(streams[0])
    for a, s in zip(coef, streams):
        total = total + a * s
    assert len(coef) == len(streams)
    return total


def gru_candidate(u):
    return torch.where(u >= 0, u + 0.5, sigmoid(u))


def gru_scan(z, cand, start=None):
    """S_t = (1 - z_t) S_(t-1) + z_t cand_t, channel by channel; S before the first token is zero or ``start``."""
    s = torch.zeros(z.shape[1], dtype=F64) if start is None else start.clone()
    out = []
    for t in range(z.shape[0]):
        s = (1.0 - z[t]) * s + z[t] * cand[t]
        out.append(s)
    return torch.stack(out)


def mingru(h, w, p):
    z = sigmoid(h @ w[p + ".z"].T + w[p + ".z.b"])
    u = h @ w[p + ".x"].T + w[p + ".x.b"]
    g = h @ w[p + ".g"].T
    s = gru_scan(z, gru_candidate(u))
    return (s * (g * sigmoid(g))) @ w[p + ".o"].T


def latent_attention(h, w, p, m, pos, eps):
    t = h.shape[0]
    H, D, R, V, KR = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    base, dims = m["rot"]["base"], m["rot"]["dims"]
    q = (h @ w[p + ".q"].T).view(t, H, D + R)
    dkv = h @ w[p + ".dkv"].T
    c = unit(dkv[:, :KR], eps) * w[p + ".dkv.norm"]
    shared_key = rotate_half(dkv[:, KR:], pos, base, dims)
    keys = (c @ w[p + ".uk"].T).view(t, H, D)
    vals = (c @ w[p + ".uv"].T).view(t, H, V)
    later = pos[None, :] > pos[:, None]
    heads = []
    for hd in range(H):
        turned = rotate_half(q[:, hd, D:], pos, base, dims)
        score = (q[:, hd, :D] @ keys[:, hd].T + turned @ shared_key.T) * m["scale"]
        score = score.masked_fill(later, -math.inf)
        heads.append(torch.softmax(score, dim=-1) @ vals[:, hd])
    return torch.cat(heads, dim=-1) @ w[p + ".o"].T


def poly_norm(z, act, eps):
    a, b, c, e = act
    return a * unit(z, eps) + b * unit(z ** 2, eps) + c * unit(z ** 3, eps) + e


def dense_ff(h, w, p, eps):
    return poly_norm(h @ w[p + ".up"].T, w[p + ".act"], eps) @ w[p + ".down"].T


def expert(h, w, p, limit):
    g = torch.clamp(h @ w[p + ".gate"].T, max=limit)
    u = torch.clamp(h @ w[p + ".up"].T, -limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ w[p + ".down"].T


def route(h, w, p, r):
    """-> per token: [(expert, score)], best first."""
    s = sigmoid(h @ w[p + ".router"].T)
    return [[(e, float(row[e])) for e in sorted(range(r["experts"]), key=lambda e: (-float(row[e]), e))[:r["top"]]]
            for row in s]


def moe_ff(h, w, p, f):
    y = torch.zeros_like(h)
    for t, picks in enumerate(route(h, w, p, f["router"])):
        for e, score in picks:
            y[t] += expert(score * h[t:t + 1], w, f"{p}.e{e}", f["expert"]["limit"])[0]
    return y


def soft_cap(x, cap):
    return cap * torch.tanh(x / cap)


def run(cfg, w, tokens):
    """(logits [T, vocab], every layer's result after its depth average [layers, T, width]) of a whole sequence."""
    eps = cfg["norm"]["eps"]
    pos = torch.arange(len(tokens))
    x = zero_norm(w["embed"][torch.tensor(tokens)], eps, w["embed.norm"])
    results, after = [x], []
    for i, layer in enumerate(cfg["layers"]):
        p, m, f = f"l{i}", layer["mixer"], layer.get("mlp")
        h = zero_norm(x, eps, w[p + ".norm1"])
        y = (mingru(h, w, p + ".mix") if layer["type"] == "mingru"
             else latent_attention(h, w, p + ".mix", m, pos, eps))
        x = x + zero_norm(y, eps, w[p + ".norm1b"])
        if f is not None:
            h = zero_norm(x, eps, w[p + ".norm2"])
            y = dense_ff(h, w, p + ".mlp", eps) if f["kind"] == "dense" else moe_ff(h, w, p + ".mlp", f)
            x = x + zero_norm(y, eps, w[p + ".norm2b"])
        results.append(x)
        x = depth_average(results, w[p + ".dwa"])
        after.append(x)
    logits = zero_norm(x, eps, w["final.norm"]) @ w["embed"].T
    if cfg.get("logit_softcap"):
        logits = soft_cap(logits, cfg["logit_softcap"])
    return logits, torch.stack(after)


def forward(cfg, w, tokens):
    return run(cfg, w, tokens)[0]


def greedy(cfg, w, prompt, n):
    ids = list(prompt)
    for _ in range(n):
        ids.append(int(forward(cfg, w, ids)[-1].argmax()))
    return ids[len(prompt):]


# --------------------------------------------------------------------------- checkpoints
def attention(heads, dim, rot_dim, vdim, kv_rank, mlp, base=10000.0, scale=None):
    return {"type": "latent_attention", "mlp": mlp,
            "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank,
                      "rot": {"base": base, "dims": rot_dim}, "scale": scale if scale is not None else (dim + rot_dim) ** -0.5}}


def gru(width, mlp):
    return {"type": "mingru", "mixer": {"width": width}, "mlp": mlp}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(ff, experts, top, limit):
    return {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "router": {"experts": experts, "top": top}}


def make_config(vocab, width, layers, softcap=20.0, eps=1e-5):
    cfg = {"architecture": "Zupilorn", "layers": layers, "norm": {"eps": eps}, "vocab": vocab, "width": width}
    if softcap:
        cfg["logit_softcap"] = softcap
    return cfg


def make_weights(cfg, seed=0):
    """bf16-representable float64 weights (what a bf16 checkpoint holds), activations of order one.  Depth averages
    mix every earlier stream in, of either sign."""
    g = torch.Generator().manual_seed(seed)

    def rnd(*shape, std=None, mean=0.0):
        t = mean + torch.randn(shape, generator=g) * (std if std is not None else shape[-1] ** -0.5)
        return t.to(torch.bfloat16).to(F64)

    wd, w = cfg["width"], {}
    w["embed"] = rnd(cfg["vocab"], wd, std=1.0)
    w["embed.norm"] = rnd(wd, std=0.3)
    for i, L in enumerate(cfg["layers"]):
        p, m, f = f"l{i}", L["mixer"], L.get("mlp")
        for n in ("norm1", "norm1b") + (("norm2", "norm2b") if f is not None else ()):
            w[f"{p}.{n}"] = rnd(wd, std=0.3)
        w[p + ".dwa"] = torch.cat([rnd(i + 1, std=0.4), rnd(1, std=0.2, mean=1.0)])
        if L["type"] == "mingru":
            n = m["width"]
            for k in ("z", "x", "g"):
                w[f"{p}.mix.{k}"] = rnd(n, wd, std=1.5 * wd ** -0.5)
            w[p + ".mix.z.b"], w[p + ".mix.x.b"] = rnd(n, std=1.5, mean=-1.5), rnd(n, std=0.5)
            w[p + ".mix.o"] = rnd(wd, n)
        else:
            H, D, R, V, KR = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
            w[p + ".mix.q"] = rnd(H * (D + R), wd, std=2.0 * wd ** -0.5)
            w[p + ".mix.dkv"], w[p + ".mix.dkv.norm"] = rnd(KR + R, wd), rnd(KR, std=0.3, mean=1.0)
            w[p + ".mix.uk"] = rnd(H * D, KR, std=2.0 * KR ** -0.5)
            w[p + ".mix.uv"] = rnd(H * V, KR)
            w[p + ".mix.o"] = rnd(wd, H * V)
        if f is None:
            continue
        if f["kind"] == "dense":
            w[p + ".mlp.up"], w[p + ".mlp.down"] = rnd(f["ff"], wd), rnd(wd, f["ff"])
            w[p + ".mlp.act"] = rnd(4, std=0.6)
        else:
            w[p + ".mlp.router"] = rnd(f["router"]["experts"], wd, std=3.0 * wd ** -0.5)
            for e in range(f["router"]["experts"]):
                for k in ("gate", "up"):
                    w[f"{p}.mlp.e{e}.{k}"] = rnd(f["expert"]["ff"], wd, std=2.0 * wd ** -0.5)
                w[f"{p}.mlp.e{e}.down"] = rnd(wd, f["expert"]["ff"])
    w["final.norm"] = rnd(wd, std=0.3)
    return w


def save_checkpoint(folder, cfg, w) -> str:
    from safetensors.torch import save_file

    folder = Path(folder)
    folder.mkdir(parents=True, exist_ok=True)
    with open(folder / "config.json", "w") as f:
        json.dump(cfg, f)
    save_file({k: v.to(torch.bfloat16).contiguous() for k, v in w.items()}, str(folder / "model.safetensors"))
    return str(folder)


def row_errors(got, want):
    """Per row: root mean square of the mean-free difference, over that of ``want`` as a whole."""
    got, want = got.to(F64), want.to(F64)
    d = got - want
    d = d - d.mean(-1, keepdim=True)
    scale = (want - want.mean(-1, keepdim=True)).pow(2).mean().sqrt()
    return d.pow(2).mean(-1).sqrt() / scale
