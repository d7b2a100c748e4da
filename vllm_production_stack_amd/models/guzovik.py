"""Guzovik: a decoder whose layers, listed one by one in the configuration, have a norm before and a norm after every
sublayer and a learned scale per channel on what a sublayer adds, ``x += rmsnorm(sublayer(rmsnorm(x))) * scale``,
first around a mixer, then around an optional feed-forward.  The stream is fp32; the norm on a sublayer's output, its
scale (folded into that norm's weight), the add and the next norm are one kernel (``ops.gated_add_rms_norm``).

A layer may run on another layer's tensors, with cache entries of its own.  The model therefore works on layer RUNS:
a run has the tensors of some layer and its own part of a pool page.

Mixers, both over a sliding window:

- ``attention``: grouped-query attention without rotation or norm on q and k.  q | k | v | gate logits come from one
  fused projection; k and v are copied to the paged pool (``ops.window_kv_write``) and the windowed-attention kernels
  read q where the projection left it, count a sink of score 0 in the softmax denominator, multiply every head by
  the sigmoid of its gate logit and write what the output projection reads.
- ``latent_attention``: ``latent_mixer.LatentAttention`` with queries projected straight from the input (q and the KV
  latent with the shared key part in one projection), no sink and no output gate.

Feed-forwards: a dense clamped gated unit, or a mixture of silu gated units (the largest router logits, weighted by
the softmax over the chosen ones) with a shared unit that every token passes.  Logits come from an output matrix of
their own.
"""

from __future__ import annotations

import torch
import torch.nn.functional as F

from .. import ops
from ..engine.config import FeedForwardSpec, LatentMixerSpec, ModelConfig, SlidingAttentionSpec
from ..ops.reference import PAGE
from ..parallel.state import get_pp, get_tp
from .batch import BatchMeta
from .latent_mixer import LatentAttention

GLU_ALPHA = 1.702   # the dense unit: g sigmoid(1.702 g) (u + 1) on clamped g and u
GLU_UP_BIAS = 1.0
ROW_RUN = 8         # rows of a fused projection are padded to whole runs of this many (16-byte rows in bf16)


class GuzovikLayer:
    """Tensors of a layer.  ``post1`` / ``post2``: (1 + weight of the norm on the sublayer's output) * layer scale."""
    __slots__ = ("spec", "norm1", "post1", "norm2", "post2", "w_in", "w_o", "sink", "dkv_norm", "w_uk", "w_uv", "w_vk",
                 "cache_offset", "cos_sin", "w_gu", "w_down", "router", "w13", "w2", "w_sh13", "w_sh2")

    def __init__(self, spec):
        for s in self.__slots__:
            setattr(self, s, None)
        self.spec = spec


class GuzovikModel(LatentAttention):
    def __init__(self, cfg: ModelConfig, dtype: torch.dtype, device: torch.device, max_model_len: int):
        if get_tp().size != 1 or get_pp().size != 1:
            raise ValueError("Guzovik runs on single-GPU replicas (no tensor / pipeline parallel layout yet)")
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError("Guzovik runs in bfloat16 or float32")
        self.cfg = cfg
        self.dtype = dtype
        self.device = device
        self.max_model_len = max_model_len
        self.specs = cfg.layer_specs
        self.n_q = cfg.num_heads
        self.n_kv = 1   # (what the runner's split count of decode rows is for: the latent layers' shared entries)
        self.head_dim = cfg.head_dim
        self.tp_size = 1
        self.lora = None
        self.layers: list[GuzovikLayer] = []   # layers that have tensors
        self.embed = self.norm = self.lm_head = None
        self.layer_probe = None  # callable(run index, fp32 residual stream after the run) for tests
        # the layer runs: (index into ``layers``, where the run's entries start inside a page, in elements)
        self.runs: list[tuple[int, int]] = []
        owners = [i for i, s in enumerate(self.specs) if s.weights_of is None]
        off = 0
        for i, s in enumerate(self.specs):
            self.runs.append((owners.index(i if s.weights_of is None else s.weights_of), off))
            m = s.mixer
            off += PAGE * (m.entry if isinstance(m, LatentMixerSpec) else m.cache_elems())
        self.page_elems = off
        self._tables: dict[tuple, torch.Tensor] = {}

    @property
    def graph_capturable(self) -> bool:
        """Decode steps can be captured when no layer's mixture falls back to the per-unit loop, which reads
        the row counts on the host (shapes the grouped GEMMs do not tile, fp32)."""
        probe = torch.empty((1, self.cfg.hidden_size), dtype=self.dtype, device=self.device)
        return self.dtype == torch.bfloat16 and self.device.type == "cuda" and all(
            lw.w13 is None or ops.moe_units_grouped(probe, lw.w13, lw.w2) for lw in self.layers)

    # ------------------------------------------------------------------ cache layout
    def kv_page_shape(self) -> tuple:
        """Shape of one page of the KV pool (the runner allocates [pages, *shape])."""
        return (self.page_elems,)

    # ------------------------------------------------------------------ weights
    def _alloc(self, gen, *shape, std=None, dtype=None, mean=0.0):
        dtype = dtype or self.dtype
        t = torch.empty(shape, dtype=torch.float32, device=self.device)
        t.normal_(mean, std if std is not None else shape[-1] ** -0.5, generator=gen)
        return t.to(dtype)

    @staticmethod
    def in_rows(m) -> dict:
        """Row ranges of a mixer's fused input projection, by the part's name; "end": its rows with padding."""
        if isinstance(m, SlidingAttentionSpec):
            parts = [("q", m.heads * m.dim), ("k", m.kv_heads * m.dim), ("v", m.kv_heads * m.vdim),
                     ("g", m.heads if m.head_gate else 0)]
        else:
            parts = [("q", m.heads * (m.dim + m.rot_dim)), ("dkv", m.entry)]
        out, at = {}, 0
        for name, n in parts:
            out[name] = (at, at + n)
            at += n
        out["end"] = (at, (at + ROW_RUN - 1) // ROW_RUN * ROW_RUN)
        return out

    def init_random(self, seed: int = 0) -> None:
        """Allocates every tensor in the layout the forward pass uses; a checkpoint overwrites them."""
        cfg = self.cfg
        w = cfg.hidden_size
        g = torch.Generator(device=self.device).manual_seed(seed)
        f32 = torch.float32

        def gain():
            return self._alloc(g, w, std=0.1, dtype=f32, mean=1.0)

        self.embed = self._alloc(g, cfg.vocab_size, w, std=1.0 / cfg.embedding_scale)
        self.layers = []
        for s in self.specs:
            if s.weights_of is not None:
                continue
            m, f = s.mixer, s.mlp
            lw = GuzovikLayer(s)
            lw.norm1, lw.post1 = gain(), gain()
            used, rows = self.in_rows(m)["end"]
            lw.w_in = self._alloc(g, rows, w)
            lw.w_in[used:] = 0
            lw.w_o = self._alloc(g, w, m.heads * m.vdim)
            if isinstance(m, SlidingAttentionSpec):
                if m.unit_sink:
                    lw.sink = torch.zeros(m.heads, dtype=f32, device=self.device)
            else:
                lw.dkv_norm = self._alloc(g, m.kv_rank, std=0.1, dtype=f32, mean=1.0)
                lw.w_uk = self._alloc(g, m.heads, m.dim, m.kv_rank)
                lw.w_uv = self._alloc(g, m.heads, m.kv_rank, m.vdim, std=m.kv_rank ** -0.5)
                lw.cos_sin = self._cos_sin(m)
            if f is not None:
                lw.norm2, lw.post2 = gain(), gain()
                if f.kind == "dense":
                    lw.w_gu = self._alloc(g, 2 * f.ff, w)
                    lw.w_down = self._alloc(g, w, f.ff)
                else:
                    lw.router = self._alloc(g, f.experts, w, dtype=f32)
                    lw.w13 = self._alloc(g, f.experts, 2 * f.ff, w)
                    lw.w2 = self._alloc(g, f.experts, w, f.ff)
                    if f.shared_ff:
                        lw.w_sh13 = self._alloc(g, 2 * f.shared_ff, w)
                        lw.w_sh2 = self._alloc(g, w, f.shared_ff)
            self.layers.append(lw)
        self.norm = gain()
        self.lm_head = self._alloc(g, cfg.vocab_size, w)

    def weight_tensors(self):
        for t in (self.embed, self.norm, self.lm_head):
            if t is not None:
                yield t
        for lw in self.layers:
            for s in GuzovikLayer.__slots__:
                t = getattr(lw, s)
                if isinstance(t, torch.Tensor) and s not in ("cos_sin", "w_vk"):
                    yield t

    def weight_bytes(self) -> int:
        return sum(t.numel() * t.element_size() for t in self.weight_tensors())

    # ------------------------------------------------------------------ batch description
    def plan_prefill(self, meta: BatchMeta, q_lens: list[int], ctx_lens: list[int], to_dev) -> None:
        self.plan_latent_prefill(meta, q_lens, ctx_lens, to_dev,
                                 [lw.spec.mixer for lw in self.layers if isinstance(lw.spec.mixer, LatentMixerSpec)])
        meta.pre_win_tiles = {}
        if self.device.type == "cuda" and self.dtype == torch.bfloat16:
            for key in sorted({(m.heads, m.kv_heads) for m in (lw.spec.mixer for lw in self.layers)
                               if isinstance(m, SlidingAttentionSpec)
                               and ops.window_mfma_supported(m.heads, m.kv_heads, m.dim, m.vdim, True)}):
                tiles = ops.build_window_tiles(q_lens, ctx_lens, *key)
                meta.pre_win_tiles[key] = torch.from_numpy(tiles).pin_memory().to(self.device, non_blocking=True)

    # ------------------------------------------------------------------ mixers
    def _attention(self, lw: GuzovikLayer, h: torch.Tensor, pool, cache_off: int, meta: BatchMeta) -> torch.Tensor:
        m: SlidingAttentionSpec = lw.spec.mixer
        rows = self.in_rows(m)
        proj = ops.linear(h, lw.w_in)  # q | k | v | gate logits
        ops.window_kv_write(proj, rows["k"][0], rows["v"][0], m.kv_heads, m.dim, m.vdim, meta.slots, pool, cache_off)
        t, nd = h.shape[0], meta.num_decode
        q = proj[:, :m.heads * m.dim].view(t, m.heads, m.dim)
        gate = proj[:, rows["g"][0]:rows["g"][1]] if m.head_gate else None
        y = torch.empty((t, m.heads, 1, m.vdim), dtype=self.dtype, device=h.device)

        def attend(a, b, block_tables, row_seq, **how):
            ops.window_attention(q[a:b], pool, cache_off, m.kv_heads, m.vdim, block_tables, row_seq, meta.positions[a:b],
                                 m.window, 0, m.scale, 0.0, lw.sink, out=y[a:b], own_values=True,
                                 head_gate=None if gate is None else gate[a:b], **how)

        if nd > 0:
            # the split count follows the batch rounded up to a power of two, which an eager step and the
            # captured step of its batch bucket share: both then sum in the same order
            attend(0, nd, meta.dec_block_tables, None,
                   splits=ops.window_decode_splits(1 << (nd - 1).bit_length(), m.kv_heads, m.window, 0, self.max_model_len))
        if meta.num_prefill_seqs > 0:
            attend(nd, t, meta.pre_block_tables, meta.pre_row_seq,
                   tiles=(meta.pre_win_tiles or {}).get((m.heads, m.kv_heads)))
        return ops.linear(y.view(t, m.heads * m.vdim), lw.w_o)

    def _latent(self, lw: GuzovikLayer, h: torch.Tensor, pool, cache_off: int, meta: BatchMeta) -> torch.Tensor:
        m: LatentMixerSpec = lw.spec.mixer
        t = h.shape[0]
        (q0, q1), (c0, c1) = self.in_rows(m)["q"], self.in_rows(m)["dkv"]
        proj = ops.linear(h, lw.w_in)  # q | KV latent | shared key part
        q = proj[:, q0:q1].view(t, m.heads, m.dim + m.rot_dim)
        ops.latent_kv_write(proj[:, c0:c1], lw.dkv_norm, meta.positions, meta.slots, lw.cos_sin, pool, cache_off, m.kv_rank,
                            m.rot_dim, m.rope_dims, self.cfg.norm_eps, q=q, q_col=m.dim)
        o = self.latent_heads(lw, q, pool, meta, cache_off)
        return ops.linear(o.view(t, m.heads * m.vdim), lw.w_o)

    # ------------------------------------------------------------------ feed-forward
    def _feed_forward(self, lw: GuzovikLayer, h: torch.Tensor) -> torch.Tensor:
        """The feed-forward's output for rows h (a mixture's in fp32)."""
        f: FeedForwardSpec = lw.spec.mlp
        if f.kind == "dense":
            return ops.linear(ops.gate_up_glu_clamp(h, lw.w_gu, f.limit, GLU_ALPHA, GLU_UP_BIAS), lw.w_down)
        logits = F.linear(h.float(), lw.router)  # a true fp32 product
        w, ids, _ = ops.route_softmax(logits, f.experts, f.experts, 1, 1, f.top, normalize=True)
        shared = ops.linear(ops.gate_up_act(h, lw.w_sh13, f.act), lw.w_sh2) if f.shared_ff else None
        ys, pos = ops.moe_units(h, lw.w13, lw.w2, ids, f.act)
        out = torch.empty(h.shape, dtype=torch.float32, device=h.device)
        return ops.moe_finish(out, ys, w, pos, shared, overwrite=True)

    # ------------------------------------------------------------------ forward
    def forward(self, input_ids: torch.Tensor, pool: torch.Tensor, meta: BatchMeta) -> torch.Tensor:
        """Final-normed hidden states of ``meta.logits_rows`` ([num_out, width], activation dtype)."""
        eps, dt = self.cfg.norm_eps, self.dtype
        x = ops.embed_scale(input_ids, self.embed, self.cfg.embedding_scale)  # fp32 residual stream
        pending: list = []  # a sublayer's output not yet in the stream, with its norm weight and a factor
        for run, (li, cache_off) in enumerate(self.runs):
            lw = self.layers[li]
            h = ops.gated_add_rms_norm(x, pending, None, None, lw.norm1, eps, dt)
            mixer = self._attention if lw.spec.type == "attention" else self._latent
            pending = [(mixer(lw, h, pool, cache_off, meta), lw.post1, 1.0)]
            if lw.spec.mlp is not None:
                h = ops.gated_add_rms_norm(x, pending, None, None, lw.norm2, eps, dt)
                pending = [(self._feed_forward(lw, h), lw.post2, 1.0)]
            if self.layer_probe is not None:
                ops.gated_add_rms_norm(x, pending, None, None, None, eps, dt, want_out=False)
                pending = []
                self.layer_probe(run, x)
        if meta.logits_rows is not None:
            x = x.index_select(0, meta.logits_rows)
            pending = [(d.index_select(0, meta.logits_rows), w, c) for d, w, c in pending]
        return ops.gated_add_rms_norm(x, pending, None, None, self.norm, eps, dt)

    def compute_logits(self, hidden: torch.Tensor) -> torch.Tensor:
        return ops.linear(hidden, self.lm_head)
