"""Cases for Zupilorn: every op against its float64 definition, and the engine on small random checkpoints
against the float64 oracle.  The CPU and the GPU test files call them with their device, dtype and tolerance."""

from __future__ import annotations

import tempfile

import torch

import zupilorn_oracle as zo
from vllm_production_stack_amd import ops
from vllm_production_stack_amd.engine.config import EngineConfig
from vllm_production_stack_amd.engine.llm_engine import LLMEngine
from vllm_production_stack_amd.engine.request import SamplingParams
from vllm_production_stack_amd.models.loader import half_to_pairs

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
    """Both mixers, both feed-forwards behind each of them, a layer of either kind without one, sizes that differ from
    one another wherever they can, two rotation bases, top 1 and top 3."""
    return zo.make_config(97, 72, [
        zo.gru(56, zo.moe(24, 6, 3, 0.8)),
        zo.attention(3, 16, 8, 24, 40, zo.dense(104), base=500.0),
        zo.gru(88, None),
        zo.attention(2, 8, 12, 16, 56, zo.moe(16, 5, 1, 1.5), base=20000.0),
        zo.gru(40, zo.dense(48)),
        zo.attention(5, 12, 4, 20, 32, None, base=500.0, scale=0.4),
    ], softcap=12.0, eps=1e-4)


def config_b():
    """Sizes that are multiples of nothing, a single head, heads of one rotated pair, every expert chosen, a single
    expert, no soft cap, attention first."""
    return zo.make_config(61, 45, [
        zo.attention(1, 5, 2, 7, 9, zo.moe(11, 4, 4, 0.5), base=77.0),
        zo.attention(4, 3, 6, 5, 23, zo.dense(33), base=9000.0, scale=1.1),
        zo.gru(29, zo.moe(13, 1, 1, 3.0)),
        zo.gru(1, zo.dense(7)),
    ], softcap=0.0, eps=1e-3)


def config_c():
    """Cache entries of 64 + 32 and 128 + 64 values (the tile kernel takes both), heads it also takes expanded for
    large prefill parts (values 64 | keys 64 + 32), units the grouped GEMMs tile and units the weight-streaming
    decode kernels take as well, a recurrence wider than one workgroup's channels."""
    return zo.make_config(200, 128, [
        zo.attention(3, 64, 32, 64, 64, zo.dense(320), base=700.0),
        zo.gru(320, zo.moe(512, 4, 2, 1.0)),
        zo.attention(2, 24, 64, 40, 128, zo.moe(64, 6, 2, 2.0), base=5000.0),
        zo.gru(130, zo.moe(128, 3, 1, 0.7)),
    ], softcap=25.0, eps=2e-6)


def config_d():
    """Recurrences only: pages hold nothing."""
    return zo.make_config(50, 40, [zo.gru(24, zo.dense(64)), zo.gru(48, zo.moe(16, 3, 2, 1.0))], softcap=9.0)


def config_e():
    """Attention only: the state slots stay empty; one layer depth and a mixture behind it."""
    return zo.make_config(53, 32, [zo.attention(2, 8, 8, 12, 24, zo.moe(16, 4, 2, 1.2))], softcap=40.0, eps=1e-6)


# ----------------------------------------------------------------------------- mechanisms
def case_embedding(dev, dtype, tol):
    dt = DTYPES[dtype]
    g = torch.Generator().manual_seed(0)
    for n in (5, 48, 300, 2056):
        table = (torch.randn(11, n, generator=g) * 0.2).to(dt)
        w = torch.randn(n, generator=g) * 0.3
        ids = torch.tensor([3, 0, 10, 3, 7])
        second = torch.full((5, n), -1.0, device=dev)
        y = ops.embed_rms_norm(ids.to(dev), table.to(dev), (1.0 + w).to(dev), 1e-3, out=second)
        want = zo.zero_norm(table[ids].double(), 1e-3, w.double())
        close(y, want, tol, f"width {n}")
        assert y.dtype == torch.float32 and torch.equal(y, second)


def case_depth_average(dev, dtype, tol):
    """The end of a layer: its last add (with and without the norm on the sublayer's output), the kept result, the
    average over every stream before it, the next norm; widths that take 16-byte loads and widths that do not."""
    dt = DTYPES[dtype]
    g = torch.Generator().manual_seed(1)
    eps, rows = 1e-4, 6
    for n in (5, 48, 300, 2304, 4104, 8200):
        for n_prev, keep, how in ((1, True, "normed"), (2, False, "fp32"), (5, True, "strided"), (4, False, "none"),
                                  (0, True, "plain"), (3, True, "fp32")):
            hist = torch.randn(n_prev + 2, rows, n, generator=g)
            res = torch.randn(rows, n, generator=g) * 2
            coef = torch.randn(n_prev + 1, generator=g)
            w = torch.rand(n, generator=g) + 0.5
            dw = None if how == "plain" else torch.rand(n, generator=g) + 0.5
            d = torch.randn(rows, n + 8, generator=g) * 3
            d = d.to(torch.float32 if how == "fp32" else dt)
            d = d[:, 8:] if how == "strided" else d[:, :n].contiguous()
            s = res.double()
            if how != "none":
                s = s + (d.double() if dw is None else zo.unit(d.double(), eps) * dw.double())
            streams = [h.double() for h in hist[:n_prev]] + [s]
            want = zo.depth_average(streams, coef.double())
            hd, rd = hist.clone().to(dev), res.clone().to(dev)
            delta = None if how == "none" else (d if how != "strided" else d._base).to(dev)
            if how == "strided":
                delta = delta[:, 8:]
            y = ops.depth_mix_rms_norm(rd, delta, None if dw is None or how == "none" else dw.to(dev), hd, n_prev, keep,
                                       coef.to(dev), w.to(dev), eps, dt)
            what = f"width {n}, {n_prev} before, {how}"
            close(rd, want, 2e-5, what)
            close(y, zo.unit(want, eps) * w.double(), tol, what + " (norm)")
            assert torch.equal(hd[:n_prev].cpu(), hist[:n_prev]) and torch.equal(hd[n_prev + 1:].cpu(), hist[n_prev + 1:])
            if keep:
                close(hd[n_prev], s, 2e-5, what + " (kept)")
            else:
                assert torch.equal(hd[n_prev].cpu(), hist[n_prev])
        rd = res.clone().to(dev)
        assert ops.depth_mix_rms_norm(rd, None, None, hd, n_prev, False, coef.to(dev), None, eps, dt, want_out=False) is None


def case_poly_norm(dev, dtype, tol):
    dt = DTYPES[dtype]
    g = torch.Generator().manual_seed(2)
    for n in (1, 7, 48, 300, 2304, 5120, 9000, 16400):
        act = torch.randn(4, generator=g)
        wide = (torch.randn(5, n + 3, generator=g) * 2).to(dt)
        wide[1] *= 0.01   # (eps matters to the cube of small values)
        wide[2, : n // 2] *= 30
        for z in (wide[:, :n].contiguous(), wide[:, 3:]):
            want = zo.poly_norm(z.double(), act.double(), 1e-5)
            zd = z.to(dev) if z.is_contiguous() else wide.to(dev)[:, 3:]
            close(ops.poly_norm(zd, act.to(dev), 1e-5), want, tol, f"{n} values")
    x = (torch.randn(6, 64, generator=g)).to(dt)
    w = (torch.randn(96, 64, generator=g) * 0.125).to(dt)
    act = torch.randn(4, generator=g)
    want = zo.poly_norm(x.double() @ w.double().T, act.double(), 1e-5)
    close(ops.up_poly_norm(x.to(dev), w.to(dev), act.to(dev), 1e-5), want, 2 * tol, "with its projection")


def case_soft_cap(dev, dtype, tol):
    dt = DTYPES[dtype]
    x = (torch.randn(3, 333, generator=torch.Generator().manual_seed(3)) * 20).to(dt)
    for cap in (3.0, 30.0):
        y = ops.soft_cap(x.to(dev), cap)
        assert y.dtype == dt
        close(y, zo.soft_cap(x.double(), cap), tol, f"cap {cap}")


def _gru_sequence(proj, off, n, zb, xb, start=None):
    z = zo.sigmoid(proj[:, off:off + n].double() + zb.double())
    cand = zo.gru_candidate(proj[:, off + n:off + 2 * n].double() + xb.double())
    gate = proj[:, off + 2 * n:off + 3 * n].double()
    s = zo.gru_scan(z, cand, None if start is None else start.double())
    return s * (gate * zo.sigmoid(gate)), s[-1]


def case_mingru(dev, dtype, tol):
    """The recurrence whole against portions down to one row (long ones cut into pieces that run side by side), slots
    that held something else, gates that hold a first token for hundreds of tokens and gates that forget at once."""
    dt = DTYPES[dtype]
    g = torch.Generator().manual_seed(4)
    for n, off, t in ((5, 3, 70), (64, 0, 150), (129, 1, 300), (130, 2, 700), (320, 0, 300), (1, 0, 20)):
        proj = (torch.randn(t, off + 3 * n + 2, generator=g) * 1.5).to(dt)
        proj[0, off + n:off + 2 * n] += 6.0           # a first token that stands out ...
        zb, xb = torch.randn(n, generator=g) - 1.0, torch.randn(n, generator=g) * 0.5
        zb[: (n + 1) // 2] -= 6.0                     # ... and channels that keep it
        want, last = _gru_sequence(proj, off, n, zb, xb)
        for chunks in ([t], [1] * min(t, 40) + [t], [2, 1, t // 2, 3, 2, t], [t - 1, 1], [128, 129, 257, t]):
            state = torch.full((3, 4 + n + 1), float("nan"), device=dev)
            state[1] = -3.0
            out, at = [], 0
            for c in chunks:
                c = min(c, t - at)
                if c <= 0:
                    continue
                rows = proj[at:at + c].contiguous().to(dev)
                cut = ops.build_gru_pieces([c]) if dev.type == "cuda" else None
                pieces = None if cut is None else tuple(torch.from_numpy(a).to(dev) for a in cut)
                y = ops.mingru_scan(rows, off, off + n, off + 2 * n, n, zb.to(dev), xb.to(dev), state, 4, i32([0, c], dev),
                                    i32([1], dev), i32(list(range(at, at + c)), dev), pieces=pieces)
                assert y.dtype == dt
                out.append(y.double().cpu())
                at += c
            close(torch.cat(out), want, tol, f"{n} channels, {len(out)} portions")
            close(state[1, 4:4 + n], last, 2e-5, f"{n} channels, end state")
            assert torch.isnan(state[[0, 2]]).all() and (state[1, :4] == -3.0).all() and state[1, -1] == -3.0


def case_mingru_batch(dev, dtype, tol):
    """Sequences side by side: single rows that go on from their slots beside chunks, one fresh and one going on, a
    long one in pieces, rows of no sequence; each in a slot of its own."""
    dt = DTYPES[dtype]
    g = torch.Generator().manual_seed(5)
    n = 70
    for lens in ([1, 1, 1, 300, 2, 513, 40], [1, 1, 1, 30, 2, 13, 40], [1, 1, 1, 1], [2, 2]):
        starts = [7, 0, 63, 0, 129, 64, 1][:len(lens)]      # position of each sequence's first row
        slots = [4, 2, -1, 0, 6, 1, 5][:len(lens)]
        total = sum(lens)
        cu = [0]
        pos = []
        for ln, p in zip(lens, starts):
            cu.append(cu[-1] + ln)
            pos += list(range(p, p + ln))
        proj = torch.randn(total, 3 * n, generator=g).to(dt)
        zb, xb = torch.randn(n, generator=g) - 2.0, torch.randn(n, generator=g) * 0.5
        held = torch.randn(8, n, generator=g)
        state = held.clone().to(dev)
        cut = ops.build_gru_pieces(lens) if dev.type == "cuda" else None
        assert dev.type != "cuda" or (cut is not None) == (max(lens) > 256)
        pieces = None if cut is None else tuple(torch.from_numpy(a).to(dev) for a in cut)
        y = ops.mingru_scan(proj.to(dev), 0, n, 2 * n, n, zb.to(dev), xb.to(dev), state, 0, i32(cu, dev), i32(slots, dev),
                            i32(pos, dev), pieces=pieces)
        untouched = set(range(8))
        for i, (ln, p, slot) in enumerate(zip(lens, starts, slots)):
            start = held[slot] if p > 0 and slot >= 0 else None
            want, last = _gru_sequence(proj[cu[i]:cu[i + 1]], 0, n, zb, xb, start)
            close(y[cu[i]:cu[i + 1]], want, tol, f"sequence {i} of {lens}")
            if slot >= 0:
                untouched.discard(slot)
                close(state[slot], last, 2e-5, f"state of sequence {i} of {lens}")
        for s in untouched:
            assert torch.equal(state[s].cpu(), held[s])


def case_routing(dev):
    g = torch.Generator().manual_seed(6)
    for experts, top in ((1, 1), (6, 1), (6, 6), (11, 3), (130, 5)):
        logits = torch.randn(33, experts, generator=g) * 2
        r = {"experts": experts, "top": top}
        want = zo.route(logits.double(), {"x.router": torch.eye(experts, dtype=F64)}, "x", r)
        w, ids, _ = ops.group_topk(logits.to(dev), experts, 1, 1, top, 1.0)
        for t in range(33):
            assert [e for e, _ in want[t]] == ids[t].tolist()
            close(w[t], torch.tensor([s for _, s in want[t]], dtype=F64), 1e-6, f"scores of token {t}")


def case_scaled_units(dev, dtype, tol, shapes):
    """A routing weight on the unit's INPUT: weights far from one, so that scaling the output instead, or scaling
    after the clamps, shows; the sum over a token's pairs has no weights left."""
    dt = DTYPES[dtype]
    g = torch.Generator().manual_seed(7)
    for hidden, inter, e, top, tokens in shapes:
        x = torch.randn(tokens, hidden, generator=g).to(dt)
        w13 = (torch.randn(e, 2 * inter, hidden, generator=g) * 2 * hidden ** -0.5).to(dt)
        w2 = (torch.randn(e, hidden, inter, generator=g) * inter ** -0.5).to(dt)
        ids = torch.stack([torch.randperm(e, generator=g)[:top] for _ in range(tokens)]).int()
        scale = torch.rand(tokens, top, generator=g) * 1.5 + 0.05
        scale[0] = 3.0
        wd = {f"e{j}.{k}": v.double() for j in range(e)
              for k, v in (("gate", w13[j, :inter]), ("up", w13[j, inter:]), ("down", w2[j]))}
        want = torch.zeros(tokens, hidden, dtype=F64)
        for t in range(tokens):
            for k in range(top):
                want[t] += zo.expert(float(scale[t, k]) * x[t:t + 1].double(), wd, f"e{int(ids[t, k])}", 1.1)[0]
        ys, pos = ops.moe_glu(x.to(dev), w13.to(dev), w2.to(dev), ids.to(dev), 1.1, scale=scale.to(dev))
        out = torch.full((tokens, hidden), 7.0, device=dev)
        ops.moe_finish(out, ys, None, pos, overwrite=True)
        close(out, want, tol, f"{hidden} x {inter}, {tokens} tokens, {top} of {e}")
        plain, pos = ops.moe_glu(x.to(dev), w13.to(dev), w2.to(dev), ids.to(dev), 1.1)   # and without a factor
        one = zo.expert(x[:1].double(), wd, f"e{int(ids[0, 0])}", 1.1)[0]
        close(plain[int(pos[0])], one, tol, "unscaled")


def case_rotation_layout(dev):
    """Query and key rows stored for pairs (i, i + dims/2), reordered at load, through the kernels that rotate
    neighbours: scores at unequal positions are those of the stored layout, also with channels that do not rotate."""
    g = torch.Generator().manual_seed(8)
    for dims, rot, width in ((8, 8, 12), (2, 2, 5), (6, 10, 16), (32, 32, 40)):
        wq, wk = torch.randn(rot, width, generator=g), torch.randn(rot, width, generator=g)
        h = torch.randn(7, width, generator=g)
        pos = torch.tensor([0, 1, 5, 63, 64, 130, 999])
        table = ops.build_cos_sin(dims, 1024, 321.0).to(dev)
        got = []
        for w in (wq, wk):
            x = (h @ half_to_pairs(w, dims).T).view(7, 1, rot).to(dev)
            ops.rope_pairs(x, pos.int().to(dev), table, 0, dims)
            got.append(x[:, 0].double().cpu())
        want = [zo.rotate_half((h @ w.T).double(), pos, 321.0, dims) for w in (wq, wk)]
        close(got[0] @ got[1].T, want[0] @ want[1].T, 2e-5, f"{dims} of {rot} channels")


# ----------------------------------------------------------------------------- the engine
def make_engine(cfg, w, device, dtype, pages=12, slots=4, budget=None, eager=True):
    folder = zo.save_checkpoint(tempfile.mkdtemp(prefix="zp-"), cfg, w)
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
    """Every row within ``tol``; with ``loose`` (16-bit runs) that many rows may miss it: a routing decision that
    rounding turns over changes a row (and, through the state, later ones), and says nothing about the kernels."""
    assert got.shape == want.shape, f"{what}: shape {tuple(got.shape)} != {tuple(want.shape)}"
    err = zo.row_errors(got, want)
    assert torch.isfinite(err).all(), what
    bad = int((err >= tol).sum())
    loose = max(loose, int(loose / 100 * got.shape[0]))   # from 100 rows on, that many per cent
    assert err.median().item() < tol and bad <= loose, \
        f"{what}: {bad} rows off, the worst (row {int(err.argmax())}) by {err.max().item():.3g} (allowed {tol})"


def check_cuts(device, dtype, tol, cfg, w, n, cuts_list, seed=1, pages=12, loose=0):
    toks = tokens(cfg, n, seed)
    want = zo.forward(cfg, w, toks)
    eng = make_engine(cfg, w, device, dtype, pages=pages)
    for k, cuts in enumerate(cuts_list):
        check_rows(replay(eng, f"r{k}", toks, cuts), want, tol, f"cuts {cuts[:6]}", loose)
    assert eng.bm.num_free() == pages and eng.scheduler.state_slots.num_free() == 4  # pages and slots came back
    eng.shutdown()


def check_layers(device, dtype, tol, cfg, w, n=37):
    """The residual stream after every layer's depth average."""
    toks = tokens(cfg, n, 5)
    logits, want = zo.run(cfg, w, toks)
    eng = make_engine(cfg, w, device, dtype)
    got = {}
    eng.runner.model.layer_probe = lambda i, x: got.__setitem__(i, x.detach().double().cpu().clone())
    out = eng.forced_step([("a", toks, [3, n - 1])], ["a"]).cpu()
    assert len(got) == want.shape[0]
    for i in range(want.shape[0]):
        err = ((got[i] - want[i]).pow(2).mean(-1).sqrt() / want[i].pow(2).mean(-1).sqrt()).median().item()
        assert err < tol, f"layer {i}: error {err:.3g}"
    check_rows(out, logits[[3, n - 1]], tol, "rows wanted beside the probe", loose=2)
    eng.shutdown()


def check_batches(device, dtype, tol, cfg, w, loose=0):
    """Unequal requests in the same steps (portions beside single tokens); pages and state slots are used
    again, by requests that start while others are in the middle of theirs; every request as if it were alone."""
    lens = [150, 3, 70, 1, 129, 66, 40]
    reqs = {f"q{i}": tokens(cfg, n, 20 + i) for i, n in enumerate(lens)}
    want = {k: zo.forward(cfg, w, v) for k, v in reqs.items()}
    pages = 8  # 512 tokens: less than the sum of all requests
    eng = make_engine(cfg, w, device, dtype, pages=pages, slots=3)
    at = {k: 0 for k in reqs}
    got = {k: [] for k in reqs}
    chunk = {"q0": [31, 2, 64, 1, 1, 33], "q1": [2], "q2": [5, 59, 2], "q3": [1], "q4": [64, 2, 61], "q5": [66],
             "q6": [3, 30]}
    live, waiting = [], list(reqs)
    used_slots = []
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
        used_slots += [r.state_slot for r in eng.scheduler.running]
        row = 0
        for k, t, _ in entries:
            got[k].append(logits[row:row + len(t)])
            row += len(t)
        live = [k for k in live if k not in end]
    for k in reqs:
        check_rows(torch.cat(got[k]), want[k], tol, f"{k} ({len(reqs[k])} tokens)", loose)
    assert eng.bm.num_free() == pages and not eng.scheduler.running and eng.scheduler.state_slots.num_free() == 3
    assert len(reqs) > 3 >= len(set(used_slots))  # seven requests went through three slots
    eng.shutdown()


def check_generate(device, dtype, cfg, w, n_new=10, eager=True):
    """Greedy generation through the engine's own entry point: scheduler, chunked prefill, sampler."""
    prompts = [tokens(cfg, n, 40 + n) for n in (90, 5, 1, 66, 30)]
    eng = make_engine(cfg, w, device, dtype, pages=10, slots=3, budget=48, eager=eager)  # prompts are cut at 48 rows
    outs = eng.generate(prompts, SamplingParams(max_tokens=n_new, temperature=0.0, ignore_eos=True))
    for p, o in zip(prompts, outs):
        assert o == zo.greedy(cfg, w, p, n_new), f"prompt of {len(p)} tokens"
    assert eng.scheduler.state_slots.num_free() == 3 and eng.bm.num_free() == 10
    eng.shutdown()


def check_preemption(device, dtype, cfg, w):
    """A pool too small for all running sequences: the scheduler preempts, the victim gives its slot and
    pages back and is recomputed from its first token; the tokens do not change."""
    prompts = [tokens(cfg, n, 70 + n) for n in (60, 61, 62)]
    n_new = 20
    eng = make_engine(cfg, w, device, dtype, pages=3, slots=3, budget=64)
    outs = eng.generate(prompts, SamplingParams(max_tokens=n_new, temperature=0.0, ignore_eos=True))
    assert eng.scheduler.num_preemptions > 0
    for p, o in zip(prompts, outs):
        assert o == zo.greedy(cfg, w, p, n_new)
    eng.shutdown()


def pointed(cfg, w, token, gain=9.0):
    """Weights under which one token stands out among hundreds.  Layer 0 latent attention: the embeddings share a
    direction that every query follows, and the token's key lies along what the queries then look for, so rows
    anywhere behind the token attend to it above all.  Layer 0 minGRU: half of the channels keep what they hold for
    hundreds of tokens, and let the token in wide open."""
    w = {k: v.clone() for k, v in w.items()}
    wd, eps = cfg["width"], cfg["norm"]["eps"]
    w["embed"] = w["embed"] + 0.5 * torch.sign(torch.arange(wd, dtype=F64) % 2 - 0.5)
    w["embed"] = w["embed"].to(torch.bfloat16).double()
    h = zo.zero_norm(zo.zero_norm(w["embed"], eps, w["embed.norm"]), eps, w["l0.norm1"])   # layer 0's input, per token
    common = h.mean(0) / h.mean(0).pow(2).sum()
    apart = h[token] - h.mean(0)
    apart = apart / (apart @ h[token])                       # 1 for the token, about 0 for the others
    m = cfg["layers"][0]["mixer"]
    if cfg["layers"][0]["type"] == "mingru":
        n = m["width"] // 2
        w["l0.mix.z.b"][:n] = -12.0
        w["l0.mix.z"][:n] = 0.1 * w["l0.mix.z"][:n] + 16.0 * apart
        w["l0.mix.x"][:n] += 6.0 * apart
    else:
        H, D, R = m["heads"], m["dim"], m["rot_dim"]
        u = zo.unit(h[token] @ w["l0.mix.dkv"][:m["kv_rank"]].T, eps)
        look = u / w["l0.mix.dkv.norm"] / u.pow(2).sum()     # 1 for the token's latent, less for any other (all are as long)
        v = torch.zeros(D, dtype=F64)
        v[0] = gain / m["scale"] ** 0.5
        for hd in range(H):
            w["l0.mix.q"][hd * (D + R):hd * (D + R) + D] += torch.outer(v, common)
            w["l0.mix.uk"][hd * D:(hd + 1) * D] += torch.outer(v, look)
    return {k: x.to(torch.bfloat16).double() for k, x in w.items()}


def check_far_token(device, dtype, cfg, w, tol, least=0.05):
    """One token far back decides the answer (``pointed`` weights for token 7): the same long prompt twice, with and
    without it.  The logits hundreds of tokens later, in a prompt's portion and decoded, differ from each other and
    match the oracle for both."""
    n = 330
    base = [t if t != 7 else 8 for t in tokens(cfg, n, 90)]
    w = pointed(cfg, w, 7)
    for where in (0, 3, 63, 64, 128):
        a, b = list(base), list(base)
        a[where], b[where] = 7, 8
        eng = make_engine(cfg, w, device, dtype, pages=12)
        rows = [n - 70, n - 2, n - 1]
        want = {"a": zo.forward(cfg, w, a)[rows], "b": zo.forward(cfg, w, b)[rows]}
        apart = zo.row_errors(want["a"], want["b"])
        assert apart.min().item() > least, f"token {where} does not stand out: {apart.tolist()}"
        for name, toks in (("a", a), ("b", b)):
            eng.forced_step([(name, toks[:200], [])], [])
            got = [eng.forced_step([(name, toks[200:n - 1], [rows[0] - 200, rows[1] - 200])], []),
                   eng.forced_step([(name, toks[n - 1:], [0])], [name])]
            got = torch.cat(got).float().cpu()
            check_rows(got, want[name], tol, f"prompt {name}, token {where}", loose=0 if tol < 1e-3 else 1)
        eng.shutdown()
