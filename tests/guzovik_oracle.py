"""Plain float64 definition of the Guzovik decoder, one function per mechanism, and makers of small random
checkpoints.  It recomputes whole sequences (no cache, no batching, keys and values expanded per head, masks and
softmax denominators written out, every expert called token by token) and shares no code with the engine; the
engine's tests compare against it."""

from __future__ import annotations

import json
import math
from pathlib import Path

import torch

F64 = torch.float64


# --------------------------------------------------------------------------- mechanisms
def logistic(z):
    return 1.0 / (1.0 + torch.exp(-z))


def over_rms(x, eps):
    return x / torch.sqrt(x.pow(2).mean(dim=-1, keepdim=True) + eps)


def stream_norm(x, w, eps):
    """The norm around sublayers: its stored weight is the gain minus one."""
    return over_rms(x, eps) * (1.0 + w)


def visible(n, window):
    """[n, n] bool: row i sees column j when j is i itself or one of the window - 1 positions before it."""
    back = torch.arange(n)[:, None] - torch.arange(n)[None, :]
    return (back >= 0) & (back < window)


def weights_with_unit_sink(score, seen):
    """exp(s) / (1 + sum exp(s)) over the seen columns (shifted by the larger of 0 and the largest score)."""
    s = score.masked_fill(~seen, -math.inf)
    top = torch.clamp(s.max(dim=-1, keepdim=True).values, min=0.0)
    e = torch.exp(s - top)
    return e / (torch.exp(-top) + e.sum(dim=-1, keepdim=True))


def weights_plain(score, seen):
    s = score.masked_fill(~seen, -math.inf)
    e = torch.exp(s - s.max(dim=-1, keepdim=True).values)
    return e / e.sum(dim=-1, keepdim=True)


def grouped_attention(h, w, p, m):
    n = h.shape[0]
    H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = h @ w[p + ".q"].T, h @ w[p + ".k"].T, h @ w[p + ".v"].T
    gate = logistic(h @ w[p + ".g"].T)                       # one number per row and head
    seen = visible(n, m["mask"]["size"])
    heads = []
    for a in range(H):
        b = a // (H // G)
        score = (q[:, a * D:(a + 1) * D] @ k[:, b * D:(b + 1) * D].T) * m["scale"]
        out = weights_with_unit_sink(score, seen) @ v[:, b * V:(b + 1) * V]
        heads.append(out * gate[:, a:a + 1])
    return torch.cat(heads, dim=1) @ w[p + ".o"].T


def turn_neighbours(x, pos, base, dims):
    """Channels (2 i, 2 i + 1) below ``dims`` turn by pos * base^(-2 i / dims); the rest pass."""
    y = x.clone()
    for i in range(dims // 2):
        angle = pos.to(F64) * base ** (-2.0 * i / dims)
        c, s = torch.cos(angle), torch.sin(angle)
        y[:, 2 * i] = x[:, 2 * i] * c - x[:, 2 * i + 1] * s
        y[:, 2 * i + 1] = x[:, 2 * i + 1] * c + x[:, 2 * i] * s
    return y


def latent_attention(h, w, p, m, eps):
    n = h.shape[0]
    H, D, R, V, K = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    pos = torch.arange(n)
    base, dims = m["rot"]["base"], m["rot"]["dims"]
    q = (h @ w[p + ".q"].T).view(n, H, D + R)
    low = h @ w[p + ".dkv"].T
    c = over_rms(low[:, :K], eps) * w[p + ".dkv.norm"]
    shared = turn_neighbours(low[:, K:], pos, base, dims)
    keys, vals = (c @ w[p + ".uk"].T).view(n, H, D), (c @ w[p + ".uv"].T).view(n, H, V)
    seen = visible(n, m["mask"]["size"])
    heads = []
    for a in range(H):
        turned = turn_neighbours(q[:, a, D:], pos, base, dims)
        score = (q[:, a, :D] @ keys[:, a].T + turned @ shared.T) * m["scale"]
        heads.append(weights_plain(score, seen) @ vals[:, a])
    return torch.cat(heads, dim=1) @ w[p + ".o"].T


def clamped_unit(h, w, p, limit):
    g = torch.clamp(h @ w[p + ".gate"].T, max=limit)
    u = torch.clamp(h @ w[p + ".up"].T, min=-limit, max=limit)
    return (g * logistic(1.702 * g) * (u + 1.0)) @ w[p + ".down"].T


def silu_unit(h, w, p):
    g = h @ w[p + ".gate"].T
    return (g * logistic(g) * (h @ w[p + ".up"].T)) @ w[p + ".down"].T


def choose(z, top):
    """z [n, experts] -> per row [(expert, weight)]: the largest logits, softmax over those alone."""
    picks = []
    for row in z:
        order = sorted(range(z.shape[1]), key=lambda e: (-float(row[e]), e))[:top]
        e = torch.exp(row[order] - row[order[0]])
        picks.append(list(zip(order, (e / e.sum()).tolist())))
    return picks


def mixture(h, w, p, f):
    y = torch.zeros_like(h)
    for t, picks in enumerate(choose(h @ w[p + ".router"].T, f["router"]["top"])):
        for e, weight in picks:
            y[t] += weight * silu_unit(h[t:t + 1], w, f"{p}.e{e}")[0]
    if f.get("shared"):
        y = y + silu_unit(h, w, p + ".shared")
    return y


def run(cfg, w, tokens):
    """(logits [T, vocab], residual stream after every layer [layers, T, width]) of a whole sequence."""
    eps = cfg["norm"]["eps"]
    x = w["embed"][torch.tensor(tokens)] * cfg["embedding"]["scale"]
    after = []
    for i, layer in enumerate(cfg["layers"]):
        src = layer.get("weights_of")
        p, m, f = f"l{i if src is None else src}", layer["mixer"], layer.get("mlp")
        h = stream_norm(x, w[p + ".norm1"], eps)
        y = (grouped_attention(h, w, p + ".mix", m) if layer["type"] == "attention"
             else latent_attention(h, w, p + ".mix", m, eps))
        x = x + stream_norm(y, w[p + ".norm1b"], eps) * w[p + ".ls1"]
        if f is not None:
            h = stream_norm(x, w[p + ".norm2"], eps)
            y = clamped_unit(h, w, p + ".mlp", f["limit"]) if f["kind"] == "dense" else mixture(h, w, p + ".mlp", f)
            x = x + stream_norm(y, w[p + ".norm2b"], eps) * w[p + ".ls2"]
        after.append(x)
    return stream_norm(x, w["final.norm"], eps) @ w["head"].T, torch.stack(after)


def forward(cfg, w, tokens):
    return run(cfg, w, tokens)[0]


def greedy(cfg, w, prompt, n):
    ids = list(prompt)
    for _ in range(n):
        ids.append(int(forward(cfg, w, ids)[-1].argmax()))
    return ids[len(prompt):]


# --------------------------------------------------------------------------- checkpoints
def attention(heads, kv_heads, dim, vdim, window, mlp, scale=None):
    return {"type": "attention", "mlp": mlp,
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "mask": {"size": window},
                      "scale": scale if scale is not None else dim ** -0.5}}


def latent(heads, dim, rot_dim, vdim, kv_rank, window, mlp, base=10000.0, scale=None):
    return {"type": "latent_attention", "mlp": mlp,
            "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank,
                      "mask": {"size": window}, "rot": {"base": base, "dims": rot_dim},
                      "scale": scale if scale is not None else (dim + rot_dim) ** -0.5}}


def again(layers, j):
    """One more layer that runs on layer j's tensors."""
    return {**layers[j], "weights_of": j}


def dense(ff, limit):
    return {"kind": "dense", "ff": ff, "limit": limit}


def moe(ff, experts, top, shared):
    f = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}
    if shared:
        f["shared"] = {"ff": shared}
    return f


def make_config(vocab, width, layers, scale=1.0, eps=1e-5):
    return {"architecture": "Guzovik", "embedding": {"scale": scale}, "layers": layers, "norm": {"eps": eps},
            "vocab": vocab, "width": width}


def make_weights(cfg, seed=0):
    """bf16-representable float64 weights (what a bf16 checkpoint holds), activations of order one; layer scales of
    either sign and of unequal size."""
    g = torch.Generator().manual_seed(seed)

    def rnd(*shape, std=None, mean=0.0):
        t = mean + torch.randn(shape, generator=g) * (std if std is not None else shape[-1] ** -0.5)
        return t.to(torch.bfloat16).to(F64)

    wd, w = cfg["width"], {}
    w["embed"] = rnd(cfg["vocab"], wd, std=1.0 / cfg["embedding"]["scale"])

    def unit(p, ff, gain):
        w[p + ".gate"], w[p + ".up"] = rnd(ff, wd, std=gain * wd ** -0.5), rnd(ff, wd, std=gain * wd ** -0.5)
        w[p + ".down"] = rnd(wd, ff)

    for i, layer in enumerate(cfg["layers"]):
        if layer.get("weights_of") is not None:
            continue
        p, m, f = f"l{i}", layer["mixer"], layer.get("mlp")
        for k in ("1", "2") if f is not None else ("1",):
            w[f"{p}.norm{k}"], w[f"{p}.norm{k}b"] = rnd(wd, std=0.3), rnd(wd, std=0.3)
            w[f"{p}.ls{k}"] = rnd(wd, std=0.4, mean=0.6)
        if layer["type"] == "attention":
            H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
            w[p + ".mix.q"], w[p + ".mix.k"] = rnd(H * D, wd, std=1.5 * wd ** -0.5), rnd(G * D, wd, std=1.5 * wd ** -0.5)
            w[p + ".mix.v"], w[p + ".mix.g"] = rnd(G * V, wd), rnd(H, wd, std=2.0 * wd ** -0.5)
        else:
            H, D, R, V, K = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
            w[p + ".mix.q"] = rnd(H * (D + R), wd, std=2.0 * wd ** -0.5)
            w[p + ".mix.dkv"], w[p + ".mix.dkv.norm"] = rnd(K + R, wd), rnd(K, std=0.3, mean=1.0)
            w[p + ".mix.uk"], w[p + ".mix.uv"] = rnd(H * D, K, std=2.0 * K ** -0.5), rnd(H * V, K)
        w[p + ".mix.o"] = rnd(wd, H * V)
        if f is None:
            continue
        if f["kind"] == "dense":
            unit(p + ".mlp", f["ff"], 2.0)
        else:
            w[p + ".mlp.router"] = rnd(f["router"]["experts"], wd, std=3.0 * wd ** -0.5)
            for e in range(f["router"]["experts"]):
                unit(f"{p}.mlp.e{e}", f["expert"]["ff"], 1.0)
            if f.get("shared"):
                unit(p + ".mlp.shared", f["shared"]["ff"], 1.0)
    w["final.norm"] = rnd(wd, std=0.3)
    w["head"] = rnd(cfg["vocab"], wd)
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
