"""Cases for Guzovik: every op against its float64 definition, and the engine on small random checkpoints
against the float64 oracle.  The CPU and the GPU test files call them with their device, dtype and tolerance."""

from __future__ import annotations

import copy
import tempfile

import torch

import guzovik_oracle as go
from vllm_production_stack_amd import ops
from vllm_production_stack_amd.engine.config import EngineConfig
from vllm_production_stack_amd.engine.llm_engine import LLMEngine
from vllm_production_stack_amd.engine.request import SamplingParams
from vllm_production_stack_amd.ops import reference

PAGE = 64
F64 = torch.float64
DTYPES = {"float32": torch.float32, "bfloat16": torch.bfloat16}


def close(got, want, tol, what=""):
    err = (got.double().cpu() - want).abs().max().item()
    lim = tol * max(1.0, want.abs().max().item())
    assert err <= lim, f"{what}: off by {err:.3g} (allowed {lim:.3g})"


def i32(x, dev):
    return torch.tensor(x, dtype=torch.int32, device=dev)


# ----------------------------------------------------------------------------- configurations
def config_a():
    """Both mixers, both feed-forwards behind each of them, a layer of either kind without one, layers that run on
    another's tensors (next to it and far from it), windows below, at and above a page."""
    layers = [
        go.attention(6, 2, 16, 24, 70, go.moe(24, 7, 3, 40)),
        go.latent(3, 16, 8, 24, 40, 45, go.dense(104, 0.8), base=500.0),
    ]
    layers.append(go.again(layers, 0))
    layers += [
        go.attention(5, 5, 12, 8, 64, None, scale=0.5),
        go.latent(2, 8, 12, 16, 56, 130, go.moe(16, 5, 1, 0), base=20000.0, scale=0.4),
        go.attention(2, 1, 20, 28, 33, go.dense(48, 3.0)),
    ]
    layers += [go.again(layers, 1), go.again(layers, 4)]
    return go.make_config(97, 72, layers, scale=3.0, eps=1e-4)


def config_b():
    """Sizes that are multiples of nothing, a single head, windows of one, two and three positions, heads of one rotated
    pair, every expert chosen, a single expert, a layer that runs on a later one's tensors, an embedding scale of 1."""
    layers = [
        go.latent(1, 5, 2, 7, 9, 3, go.moe(11, 4, 4, 9), base=77.0),
        go.attention(4, 2, 3, 5, 65, go.moe(13, 1, 1, 6), scale=1.1),
        None,
        go.attention(1, 1, 6, 1, 1, go.dense(33, 0.5)),
        go.latent(4, 3, 6, 5, 23, 61, go.dense(7, 2.0), base=9000.0),
        go.attention(3, 1, 7, 9, 2, None),
    ]
    layers[2] = go.again(layers, 4)
    return go.make_config(61, 45, layers, scale=1.0, eps=1e-3)


def config_c():
    """Shapes the matrix-core kernels tile: window attention with 64- and 96-channel keys and 64-, 96- and 128-channel
    values, cache entries of 64 + 32 and 128 + 64 values, heads that are expanded for large prefill parts (values 64 |
    keys 64 + 32), units the grouped GEMMs tile and units the weight-streaming decode kernels take as well."""
    layers = [
        go.attention(4, 2, 64, 64, 100, go.moe(512, 4, 2, 256)),
        go.latent(3, 64, 32, 64, 64, 150, go.dense(320, 1.5), base=700.0),
        go.attention(6, 3, 96, 192, 64, go.moe(64, 6, 2, 128)),
        go.latent(2, 24, 64, 40, 128, 333, None, base=5000.0),
        go.attention(8, 2, 64, 128, 200, go.moe(128, 3, 1, 0)),
    ]
    layers += [go.again(layers, 0), go.again(layers, 1)]
    return go.make_config(200, 128, layers, scale=5.0, eps=2e-6)


def config_one(kind, window):
    """A single layer without a feed-forward: a row's logits depend on the tokens of its window alone."""
    layer = (go.attention(4, 2, 16, 12, window, None) if kind == "attention"
             else go.latent(3, 16, 8, 12, 24, window, None, base=300.0))
    return go.make_config(53, 32, [layer], scale=2.0, eps=1e-6)


def steady(cfg):
    """The same configuration with every unit of a mixture chosen: no routing decision that rounding could turn over."""
    cfg = copy.deepcopy(cfg)
    for layer in cfg["layers"]:
        if (layer.get("mlp") or {}).get("kind") == "moe":
            layer["mlp"]["router"]["top"] = layer["mlp"]["router"]["experts"]
    return cfg


# ----------------------------------------------------------------------------- mechanisms
def case_residual(dev, dtype, tol):
    """x + norm(sublayer output) * scale and the next norm, with the stored weights as the loader folds them: the norm's
    gain 1 + w times the layer scale."""
    dt = DTYPES[dtype]
    g = torch.Generator().manual_seed(0)
    eps = 1e-4
    for n in (5, 48, 300, 2304):
        x = torch.randn(6, n, generator=g) * 2
        y = (torch.randn(6, n, generator=g) * 3).to(dt)
        w, ls, nxt = (torch.randn(n, generator=g) * 0.4 for _ in range(3))
        want = x.double() + go.stream_norm(y.double(), w.double(), eps) * ls.double()
        xd = x.clone().to(dev)
        h = ops.gated_add_rms_norm(xd, [(y.to(dev), ((1 + w) * ls).to(dev), 1.0)], None, None, (1 + nxt).to(dev), eps, dt)
        close(xd, want, 2e-5, f"stream, width {n}")
        close(h, go.stream_norm(want, nxt.double(), eps), tol, f"next norm, width {n}")
        assert h.dtype == dt


def paged(dev, dt, lens, page_elems, seed=1):
    """A pool of shuffled pages, some more than the sequences need, filled with numbers of another request."""
    g = torch.Generator().manual_seed(seed)
    need = [(n + PAGE - 1) // PAGE for n in lens]
    order = torch.randperm(sum(need) + 3, generator=g).tolist()
    width = max(need)
    tables = torch.zeros(len(lens), width, dtype=torch.int32)
    at = 0
    for i, n in enumerate(need):
        tables[i, :n] = torch.tensor(order[at:at + n], dtype=torch.int32)
        at += n
    pool = (torch.randn(len(order), page_elems, generator=g) * 50).to(dt).to(dev)
    return pool, tables


def slots_of(tables, seq, positions):
    return torch.tensor([int(tables[seq, p // PAGE]) * PAGE + p % PAGE for p in positions], dtype=torch.int64)


def case_kv_write(dev, dtype):
    """Keys and values land where ``window_attention`` reads them, bit for bit; rows without a slot and everything else
    in the pool stay as they are.  Odd and 16-byte-aligned shapes, rows of several sequences, more rows than a tile."""
    dt = DTYPES[dtype]
    g = torch.Generator().manual_seed(2)
    for kv, dim, vdim, lead, off, tail in ((2, 16, 24, 32, 64, 8), (1, 5, 3, 7, 0, 1), (3, 64, 64, 128, 128, 0),
                                           (2, 40, 130, 80, 64, 4), (1, 1, 1, 2, 0, 0)):
        elems = ops.window_cache_elems(kv, dim, vdim)
        pool, tables = paged(dev, dt, [150, 70, 1], off + elems + 64)
        rows = [(0, p) for p in range(3, 140)] + [(1, p) for p in range(60, 70)] + [(2, 0)]
        slots = torch.cat([slots_of(tables, s, [p]) for s, p in rows])
        slots[5] = slots[100] = -1
        proj = torch.randn(len(rows), lead + kv * (dim + vdim) + tail, generator=g).to(dt)
        before = pool.clone().cpu()
        ops.window_kv_write(proj.to(dev), lead, lead + kv * dim, kv, dim, vdim, slots.to(dev), pool, off)
        after = pool.cpu()
        kc, vc = reference.window_cache_views(after, off, kv, dim, vdim)
        kb, vb = reference.window_cache_views(before, off, kv, dim, vdim)
        for r in range(len(rows)):
            if slots[r] < 0:
                continue
            pg, at = int(slots[r]) // PAGE, int(slots[r]) % PAGE
            assert torch.equal(kc[pg, at].reshape(-1), proj[r, lead:lead + kv * dim]), (kv, dim, vdim, r)
            assert torch.equal(vc[pg, at].reshape(-1), proj[r, lead + kv * dim:lead + kv * (dim + vdim)]), (kv, dim, vdim, r)
            kb[pg, at], vb[pg, at] = kc[pg, at], vc[pg, at]
        assert torch.equal(before, after)


def case_sliding_attention(dev, dtype, tol, shapes):
    """Sequences side by side, prompts' portions (plain and tiled) and single rows (one and several key ranges), q and
    gate logits read from a wider projection.  One key stands out: each query row of a chosen set sees it just inside its
    window, and the next one just outside; some heads see nothing but weak keys, so that the sink takes most."""
    dt = DTYPES[dtype]
    g = torch.Generator().manual_seed(3)
    for heads, kv, dim, vdim, window in shapes:
        lens = [window + 150, 40, 64, window + 1, 1]
        nq, nk, nv = heads * dim, kv * dim, kv * vdim
        cols = (nq + nk + nv + heads + 7) // 8 * 8
        elems = ops.window_cache_elems(kv, dim, vdim)
        pool, tables = paged(dev, dt, lens, 64 + elems)
        scale = dim ** -0.5
        sink = torch.zeros(heads, device=dev)
        want, projs = [], []
        for i, n in enumerate(lens):
            p = torch.randn(n, cols, generator=g)
            p[:, :nq] *= 0.5
            mark = min(n - 1, 9)                       # this token's keys answer every query's first channel
            p[:, :nq].view(n, heads, dim)[:, :, 0] = 3.0 * dim ** 0.25
            p[:, nq:nq + nk].view(n, kv, dim)[:, :, 0] = -3.0 * dim ** 0.25    # the others push the weight to the sink
            p[mark, nq:nq + nk].view(kv, dim)[:, 0] = 3.0 * dim ** 0.25
            p[mark, nq + nk:nq + nk + nv] += 4.0
            p = p.to(dt)
            pd = p.double()
            seen = go.visible(n, window)
            out = []
            for h in range(heads):
                b = h // (heads // kv)
                sc = pd[:, h * dim:(h + 1) * dim] @ pd[:, nq + b * dim:nq + (b + 1) * dim].T * scale
                o = go.weights_with_unit_sink(sc, seen) @ pd[:, nq + nk + b * vdim:nq + nk + (b + 1) * vdim]
                out.append(o * go.logistic(pd[:, nq + nk + nv + h])[:, None])
            full = torch.stack(out, dim=1)
            if n > mark + window:
                inside, outside = full[mark + window - 1], full[mark + window]
                assert inside.abs().mean() > 3 * outside.abs().mean(), "the marked key does not stand out"
            want.append(full)
            projs.append(p)
            ops.window_kv_write(p.to(dev), nq, nq + nk, kv, dim, vdim, slots_of(tables, i, range(n)).to(dev), pool, 64)

        def attend(picks, row_seq, **how):
            rows = torch.stack([projs[s][p] for s, p in picks]).to(dev)
            q = rows[:, :nq].view(len(picks), heads, dim)
            out = torch.full((len(picks), heads, 1, vdim), float("nan"), dtype=dt, device=dev)
            bt = tables if row_seq is not None else tables[[s for s, _ in picks]]
            ops.window_attention(q, pool, 64, kv, vdim, bt.to(dev).contiguous(), row_seq, i32([p for _, p in picks], dev),
                                 window, 0, scale, 0.0, sink, out=out, own_values=True,
                                 head_gate=rows[:, nq + nk + nv:nq + nk + nv + heads], **how)
            ref = torch.stack([want[s][p] for s, p in picks])
            close(out[:, :, 0], ref, tol, f"{heads}/{kv} heads, {dim}/{vdim}, window {window}, {how.keys()}")

        # single rows: first tokens, page borders, the marked key inside and outside, the last row
        picks = [(s, p) for s, n in enumerate(lens) for p in sorted({0, 1, 62, 63, 64, 65, 127, 128, n - 1, window - 1, window,
                                                                      9 + window - 1, 9 + window}) if 0 <= p < n]
        for splits in (1, 2, 3, 8):
            attend(picks, None, splits=splits)
        # portions of prompts: from the middle of a page, two rows, one sequence whole
        q_lens = [window + 110, 40, 2, window + 1, 1]
        picks = [(s, p) for s, n in enumerate(q_lens) for p in range(lens[s] - n, lens[s])]
        row_seq = i32([s for s, _ in picks], dev)
        attend(picks, row_seq)
        if dev.type == "cuda" and dt == torch.bfloat16 and ops.window_mfma_supported(heads, kv, dim, vdim, True):
            tiles = torch.from_numpy(ops.build_window_tiles(q_lens, lens, heads, kv)).to(dev)
            attend(picks, row_seq, tiles=tiles)


def case_latent_window(dev, dtype, tol, shapes):
    """Latent attention over a sliding window: single rows (one and several key ranges), prompts' portions plain and
    tiled; one entry stands out, just inside and just outside; the window that no context reaches is the whole context."""
    dt = DTYPES[dtype]
    g = torch.Generator().manual_seed(4)
    for heads, rank, rot, window in shapes:
        reach = min(window, 400)
        lens = [reach + 150, 40, 64, reach + 1, 1]
        entry = rank + rot
        pool, tables = paged(dev, dt, lens, 64 + PAGE * entry)
        view = reference.latent_cache_view(pool, 64, entry)
        scale = entry ** -0.5
        want, qs = [], []
        for i, n in enumerate(lens):
            e = torch.randn(n, entry, generator=g)
            q = torch.randn(n, heads, entry, generator=g) * 0.5
            q[:, :, 0] = 3.0 * entry ** 0.25
            e[:, 0] = -1.0
            mark = min(n - 1, 9)
            e[mark, 0] = 4.0 * entry ** 0.25
            e[mark, 1:rank] += 4.0
            e, q = e.to(dt), q.to(dt)
            sl = slots_of(tables, i, range(n))
            view[(sl // PAGE).to(dev), (sl % PAGE).to(dev)] = e.to(dev)
            seen = go.visible(n, window)
            out = [go.weights_plain(q[:, h].double() @ e.double().T * scale, seen) @ e[:, :rank].double() for h in range(heads)]
            full = torch.stack(out, dim=1)
            if n > mark + window:
                inside, outside = full[mark + window - 1, :, 1:], full[mark + window, :, 1:]
                assert inside.abs().mean() > 3 * outside.abs().mean(), "the marked entry does not stand out"
            want.append(full)
            qs.append(q)

        def attend(picks, row_seq, **how):
            q = torch.stack([qs[s][p] for s, p in picks]).to(dev)
            bt = tables if row_seq is not None else tables[[s for s, _ in picks]]
            out = ops.latent_attention(q[:, :, :rank], q[:, :, rank:], pool, 64, bt.to(dev).contiguous(), row_seq,
                                       i32([p for _, p in picks], dev), None, scale, window=window, **how)
            ref = torch.stack([want[s][p] for s, p in picks])
            close(out, ref, tol, f"{heads} heads, {rank} + {rot}, window {window}, {how.keys()}")

        picks = [(s, p) for s, n in enumerate(lens) for p in sorted({0, 1, 62, 63, 64, 65, 127, 128, n - 1, window - 1, window,
                                                                      9 + window - 1, 9 + window}) if 0 <= p < n]
        for splits in (1, 2, 3, 8):
            attend(picks, None, splits=splits)
        q_lens = [reach + 110, 40, 2, reach + 1, 1]
        picks = [(s, p) for s, n in enumerate(q_lens) for p in range(lens[s] - n, lens[s])]
        row_seq = i32([s for s, _ in picks], dev)
        attend(picks, row_seq)
        if dev.type == "cuda" and dt == torch.bfloat16 and ops.latent_mfma_supported(rank, rot):
            attend(picks, row_seq, tiles=torch.from_numpy(ops.build_latent_tiles(q_lens, lens, heads)).to(dev))


def case_expanded_entries(dev, shapes):
    """Value | key entries of single heads on the tile kernel (bf16): scores from the key alone, windows, first tokens."""
    dt = torch.bfloat16
    g = torch.Generator().manual_seed(5)
    for vdim, kdim, window in shapes:
        heads, lens, q_lens = 2, [200, 70], [130, 70]
        entry = vdim + kdim
        pool, tables = paged(dev, dt, [n for n in lens for _ in range(heads)], PAGE * entry)
        view = reference.latent_cache_view(pool, 0, entry)
        q = torch.randn(sum(q_lens), heads, kdim, generator=g).to(dt)
        want = torch.zeros(sum(q_lens), heads, vdim, dtype=F64)
        tiles, row = [], 0
        for i, (n, ctx) in enumerate(zip(q_lens, lens)):
            seen = go.visible(ctx, window)[ctx - n:]
            for h in range(heads):
                e = (torch.randn(ctx, entry, generator=g) * 1.5).to(dt)
                sl = slots_of(tables, i * heads + h, range(ctx))
                view[(sl // PAGE).to(dev), (sl % PAGE).to(dev)] = e.to(dev)
                sc = q[row:row + n, h].double() @ e[:, vdim:].double().T * 0.11
                want[row:row + n, h] = go.weights_plain(sc, seen) @ e[:, :vdim].double()
                tiles += [[i * heads + h, row + k, min(64, n - k), ctx - n + k, h, 1] for k in range(0, n, 64)]
            row += n
        pos = [p for n, ctx in zip(q_lens, lens) for p in range(ctx - n, ctx)]
        out = torch.full((sum(q_lens), heads, vdim), float("nan"), dtype=dt, device=dev)
        ops.latent_attention(None, q.to(dev), pool, 0, tables.to(dev), None, i32(pos, dev), None, 0.11, out=out,
                             tiles=i32(tiles, dev), window=window)
        close(out, want, 2e-2, f"{vdim} | {kdim}, window {window}")


def case_routing(dev):
    """The softmax over the chosen logits alone, also where they are far from zero and far from each other."""
    g = torch.Generator().manual_seed(6)
    for experts, top in ((1, 1), (6, 1), (6, 6), (11, 3), (130, 5)):
        logits = torch.randn(33, experts, generator=g) * 2
        logits[1] += 300.0
        logits[2] *= 30.0
        logits[3] -= 500.0
        want = go.choose(logits.double(), top)
        w, ids, _ = ops.route_softmax(logits.to(dev), experts, experts, 1, 1, top, normalize=True)
        for t in range(33):
            if t == 2:   # (scores that underflow next to the largest weigh nothing, whichever are chosen)
                got = dict(zip(ids[t].tolist(), w[t].tolist()))
                assert all(abs(got.get(e, 0.0) - s) < 1e-6 for e, s in want[t])
                continue
            assert [e for e, _ in want[t]] == ids[t].tolist()
            close(w[t], torch.tensor([s for _, s in want[t]], dtype=F64), 1e-6, f"weights of token {t}")


def case_mixture(dev, dtype, tol, shapes):
    """Units, their weighted sum and the shared unit, which is added as it is."""
    dt = DTYPES[dtype]
    g = torch.Generator().manual_seed(7)
    for hidden, inter, experts, top, tokens, shared in shapes:
        x = torch.randn(tokens, hidden, generator=g).to(dt)

        def stack(n, ff):
            return ((torch.randn(n, 2 * ff, hidden, generator=g) * 1.5 * hidden ** -0.5).to(dt),
                    (torch.randn(n, hidden, ff, generator=g) * ff ** -0.5).to(dt))

        w13, w2 = stack(experts, inter)
        s13, s2 = stack(1, shared or 8)
        wd = {f"e{j}.{k}": v.double() for j in range(experts)
              for k, v in (("gate", w13[j, :inter]), ("up", w13[j, inter:]), ("down", w2[j]))}
        wd.update({"shared.gate": s13[0, :shared].double(), "shared.up": s13[0, shared:].double(), "shared.down": s2[0].double()})
        logits = torch.randn(tokens, experts, generator=g) * 2
        want = torch.zeros(tokens, hidden, dtype=F64)
        for t, picks in enumerate(go.choose(logits.double(), top)):
            for e, weight in picks:
                want[t] += weight * go.silu_unit(x[t:t + 1].double(), wd, f"e{e}")[0]
        if shared:
            want += go.silu_unit(x.double(), wd, "shared")
        w, ids, _ = ops.route_softmax(logits.to(dev), experts, experts, 1, 1, top, normalize=True)
        ys, pos = ops.moe_units(x.to(dev), w13.to(dev), w2.to(dev), ids)
        sh = ops.linear(ops.gate_up_act(x.to(dev), s13[0].to(dev), "silu"), s2[0].to(dev)) if shared else None
        out = torch.full((tokens, hidden), 7.0, device=dev)
        ops.moe_finish(out, ys, w, pos, sh, overwrite=True)
        close(out, want, tol, f"{hidden} x {inter}, {tokens} tokens, {top} of {experts}, shared {shared}")


def case_clamped_unit(dev, dtype, tol):
    dt = DTYPES[dtype]
    g = torch.Generator().manual_seed(8)
    for hidden, ff, rows, limit in ((24, 40, 9, 0.7), (7, 5, 3, 2.0), (128, 320, 70, 1.3)):
        x = torch.randn(rows, hidden, generator=g).to(dt)
        wgu = (torch.randn(2 * ff, hidden, generator=g) * 2.5 * hidden ** -0.5).to(dt)
        wdn = (torch.randn(hidden, ff, generator=g) * ff ** -0.5).to(dt)
        wd = {"m.gate": wgu[:ff].double(), "m.up": wgu[ff:].double(), "m.down": wdn.double()}
        want = go.clamped_unit(x.double(), wd, "m", limit)
        y = ops.linear(ops.gate_up_glu_clamp(x.to(dev), wgu.to(dev), limit), wdn.to(dev))
        close(y, want, tol, f"{hidden} -> {ff}, limit {limit}")


# ----------------------------------------------------------------------------- the engine
def make_engine(cfg, w, device, dtype, pages=12, slots=4, budget=None, eager=True):
    folder = go.save_checkpoint(tempfile.mkdtemp(prefix="gz-"), cfg, w)
    ec = EngineConfig(model=folder, dtype=dtype, device=device, max_model_len=pages * PAGE, max_num_seqs=slots,
                      max_num_batched_tokens=budget or pages * PAGE, num_gpu_blocks_override=pages,
                      enable_prefix_caching=True, enforce_eager=eager, capture_graphs_at_start=False)
    return LLMEngine(ec)


def tokens(cfg, n, seed):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, cfg["vocab"], (n,), generator=g).tolist()


def replay(engine, rid, toks, cuts, end=True):
    """Feed ``toks`` in portions of the sizes ``cuts`` (the rest one by one), all rows wanted -> logits [T, vocab]."""
    out, at = [], 0
    sizes = list(cuts)
    while at < len(toks):
        n = min(sizes.pop(0) if sizes else 1, len(toks) - at)
        last = at + n == len(toks)
        out.append(engine.forced_step([(rid, toks[at:at + n], list(range(n)))], [rid] if last and end else []))
        at += n
    return torch.cat(out).float().cpu()


def check_rows(got, want, tol, what, loose=0):
    """Every row within ``tol``; with ``loose`` (16-bit runs) that many rows, or from 100 rows on that many per cent, may
    miss it: a routing decision that rounding turns over changes a row and says nothing about the kernels."""
    assert got.shape == want.shape, f"{what}: shape {tuple(got.shape)} != {tuple(want.shape)}"
    err = go.row_errors(got, want)
    assert torch.isfinite(err).all(), what
    bad = int((err >= tol).sum())
    loose = max(loose, int(loose / 100 * got.shape[0]))
    assert err.median().item() < tol and bad <= loose, \
        f"{what}: {bad} rows off, the worst (row {int(err.argmax())}) by {err.max().item():.3g} (allowed {tol})"


def check_cuts(device, dtype, tol, cfg, w, n, cuts_list, seed=1, pages=12, loose=0):
    toks = tokens(cfg, n, seed)
    want = go.forward(cfg, w, toks)
    eng = make_engine(cfg, w, device, dtype, pages=pages)
    for k, cuts in enumerate(cuts_list):
        check_rows(replay(eng, f"r{k}", toks, cuts), want, tol, f"cuts {cuts[:6]}", loose)
    assert eng.bm.num_free() == pages
    eng.shutdown()


def check_layers(device, dtype, tol, cfg, w, n=37):
    """The residual stream after every layer."""
    toks = tokens(cfg, n, 5)
    logits, want = go.run(cfg, w, toks)
    eng = make_engine(cfg, w, device, dtype)
    got = {}
    eng.runner.model.layer_probe = lambda i, x: got.__setitem__(i, x.detach().double().cpu().clone())
    out = eng.forced_step([("a", toks, [3, n - 1])], ["a"]).cpu()
    assert len(got) == want.shape[0]
    for i in range(want.shape[0]):
        err = ((got[i] - want[i]).pow(2).mean(-1).sqrt() / want[i].pow(2).mean(-1).sqrt()).median().item()
        assert err < tol, f"layer {i}: error {err:.3g}"
    check_rows(out, logits[[3, n - 1]], tol, "rows wanted beside the probe", loose=0 if tol < 1e-3 else 2)
    eng.shutdown()


def check_batches(device, dtype, tol, cfg, w, loose=0):
    """Unequal requests in the same steps (portions beside single tokens); pages are used again, by requests that start
    while others are in the middle of theirs; every request as if it were alone."""
    lens = [150, 3, 70, 1, 129, 66, 40]
    reqs = {f"q{i}": tokens(cfg, n, 20 + i) for i, n in enumerate(lens)}
    want = {k: go.forward(cfg, w, v) for k, v in reqs.items()}
    pages = 8  # 512 tokens: less than the sum of all requests
    eng = make_engine(cfg, w, device, dtype, pages=pages, slots=3)
    at = {k: 0 for k in reqs}
    got = {k: [] for k in reqs}
    chunk = {"q0": [31, 2, 64, 1, 1, 33], "q1": [2], "q2": [5, 59, 2], "q3": [1], "q4": [64, 2, 61], "q5": [66],
             "q6": [3, 30]}
    live, waiting = [], list(reqs)
    guard = 0
    while live or waiting:
        guard += 1
        assert guard < 400
        while waiting and len(live) < 3:
            need = (len(reqs[waiting[0]]) + PAGE - 1) // PAGE
            held = sum((len(reqs[k]) + PAGE - 1) // PAGE for k in live)
            if held + need > pages:
                break
            live.append(waiting.pop(0))
        entries, end = [], []
        for k in live:
            if len(live) > 1 and guard % 5 == 0 and k == live[0]:
                continue  # a request sits a step out and goes on later
            n = min(chunk[k].pop(0) if chunk[k] else 1, len(reqs[k]) - at[k])
            entries.append((k, reqs[k][at[k]:at[k] + n], list(range(n))))
            at[k] += n
            if at[k] == len(reqs[k]):
                end.append(k)
        logits = eng.forced_step(entries, end).float().cpu()
        row = 0
        for k, t, _ in entries:
            got[k].append(logits[row:row + len(t)])
            row += len(t)
        live = [k for k in live if k not in end]
    for k in reqs:
        check_rows(torch.cat(got[k]), want[k], tol, f"{k} ({len(reqs[k])} tokens)", loose)
    assert eng.bm.num_free() == pages and not eng.scheduler.running
    eng.shutdown()


def check_generate(device, dtype, cfg, w, n_new=10, eager=True):
    """Greedy generation through the engine's own entry point: scheduler, chunked prefill, sampler; then once more, with
    the prompts' pages found in the prefix cache."""
    prompts = [tokens(cfg, n, 40 + n) for n in (90, 5, 1, 66, 130)]
    eng = make_engine(cfg, w, device, dtype, pages=14, slots=3, budget=48, eager=eager)  # prompts are cut at 48 rows
    params = SamplingParams(max_tokens=n_new, temperature=0.0, ignore_eos=True)
    want = [go.greedy(cfg, w, p, n_new) for p in prompts]
    for again in (False, True):
        hits = eng.bm.hits
        outs = eng.generate(prompts, params)
        for p, o, ref in zip(prompts, outs, want):
            assert o == ref, f"prompt of {len(p)} tokens, second time: {again}"
        assert again == (eng.bm.hits > hits)
    assert eng.bm.num_free() == 14
    eng.shutdown()


def check_preemption(device, dtype, cfg, w):
    """A pool too small for all running sequences: the scheduler preempts, the victim gives its pages back and is
    recomputed; the tokens do not change."""
    prompts = [tokens(cfg, n, 70 + n) for n in (60, 61, 62)]
    n_new = 20
    eng = make_engine(cfg, w, device, dtype, pages=3, slots=3, budget=64)
    outs = eng.generate(prompts, SamplingParams(max_tokens=n_new, temperature=0.0, ignore_eos=True))
    assert eng.scheduler.num_preemptions > 0
    for p, o in zip(prompts, outs):
        assert o == go.greedy(cfg, w, p, n_new)
    eng.shutdown()


def pointed(cfg, w, token, gain=9.0):
    """Weights of a one-layer model under which one token stands out: the embeddings share a direction that every query
    follows, and the token's key lies along what the queries then look for, so every row whose window holds the token
    attends to it above all."""
    w = {k: v.clone() for k, v in w.items()}
    wd, eps = cfg["width"], cfg["norm"]["eps"]
    common = 0.5 * torch.sign(torch.arange(wd, dtype=F64) % 2 - 0.5) / cfg["embedding"]["scale"]
    w["embed"] = (w["embed"] + common).to(torch.bfloat16).double()
    h = go.stream_norm(w["embed"] * cfg["embedding"]["scale"], w["l0.norm1"], eps)      # layer 0's input, per token
    follow = h.mean(0) / h.mean(0).pow(2).sum()
    m = cfg["layers"][0]["mixer"]
    D = m["dim"]
    v = torch.zeros(D, dtype=F64)
    v[0] = gain / m["scale"] ** 0.5
    if cfg["layers"][0]["type"] == "attention":
        apart = h[token] - h.mean(0)
        apart = apart / (apart @ h[token])                   # 1 for the token, about 0 for the others
        for a in range(m["heads"]):
            w["l0.mix.q"][a * D:(a + 1) * D] += torch.outer(v, follow)
        for b in range(m["kv_heads"]):
            w["l0.mix.k"][b * D:(b + 1) * D] += torch.outer(v, apart)
        w["l0.mix.v"] += 4.0 * torch.outer(torch.ones(w["l0.mix.v"].shape[0], dtype=F64), apart)
        w["l0.mix.g"] = w["l0.mix.g"] * 0.2
    else:
        R = m["rot_dim"]
        u = go.over_rms(h[token] @ w["l0.mix.dkv"][:m["kv_rank"]].T, eps)
        look = u / w["l0.mix.dkv.norm"] / u.pow(2).sum()     # 1 for the token's latent, less for any other (all are as long)
        for a in range(m["heads"]):
            w["l0.mix.q"][a * (D + R):a * (D + R) + D] += torch.outer(v, follow)
            w["l0.mix.uk"][a * D:(a + 1) * D] += torch.outer(v, look)
    return {k: x.to(torch.bfloat16).double() for k, x in w.items()}


def check_window_edges(device, dtype, tol, kind, window, least=0.05):
    """The same prompt with and without a token that decides the answer (``pointed`` weights for token 7).  The last row
    whose window holds it differs and the next one does not, in a prompt's portion and decoded, wherever the token lies
    in its page; all rows match the oracle."""
    cfg = config_one(kind, window)
    w = pointed(cfg, go.make_weights(cfg, seed=6), 7)
    for where in (0, 3, 63, 64, 100):
        last = where + window - 1
        n = last + 5
        base = [t if t not in (7, 8) else 9 for t in tokens(cfg, n, 90)]
        a, b = list(base), list(base)
        a[where], b[where] = 7, 8
        rows = sorted({where, where + window // 2, last - 1, last, last + 1, last + 3} & set(range(where, n)))
        out = {}
        for name, toks in (("a", a), ("b", b)):
            want = go.forward(cfg, w, toks)[rows]
            eng = make_engine(cfg, w, device, dtype, pages=12)
            got = {"prompt": replay(eng, "p", toks, [n])[rows],
                   "portions": replay(eng, "q", toks, [max(1, where), 2, max(1, window - 3), 2])[rows],
                   "decoded": replay(eng, "r", toks, [min(where + 1, n - 1)])[rows]}
            eng.shutdown()
            for how, g in got.items():
                check_rows(g, want, tol, f"{kind}, window {window}, token {where}, {how}, {name}", loose=0 if tol < 1e-3 else 1)
            out[name] = got
        for how in out["a"]:
            apart = go.row_errors(out["a"][how], out["b"][how])
            for r, e in zip(rows, apart.tolist()):
                if r <= last:
                    assert e > least, f"{kind}, window {window}, token {where}, row {r}, {how}: the token is not seen"
                else:
                    assert e < 1e-6, f"{kind}, window {window}, token {where}, row {r}, {how}: a token outside is seen"
