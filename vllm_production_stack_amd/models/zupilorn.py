"""Zupilorn: a decoder whose layers, listed one by one in the configuration, mix tokens by latent attention or by a
gated recurrence, and whose residual stream is a learned average over the depth.

Every sublayer has a norm before and a norm after it, ``x += rmsnorm(sublayer(rmsnorm(x)))``, first around a mixer,
then around an optional feed-forward; the stream is fp32.  The embedding output (RMS-normed table rows) and every
layer's result stay in a history of streams for the step, and what goes on to the next layer (and to the output) is
a weighted sum of all of them (``ops.depth_mix_rms_norm``, fused with the layer's last add and the next norm).

Mixers:

- ``mingru``: gates and candidate of a recurrence from the current token only (z | x | g in one projection), one
  fp32 state value per channel in the sequence's slot, the output gated by silu (``ops.mingru_scan``).
- ``latent_attention``: ``latent_mixer.LatentAttention`` with queries projected straight from the input (q and the KV
  latent with the shared key part in one projection), no sink and no output gate.  The checkpoint rotates channels
  (i, i + dims / 2); query and key rows are reordered at load so that partners are neighbours.

Feed-forwards: a dense one with the PolyNorm activation, or a mixture of clamped gated units chosen by sigmoid
scores, whose weight multiplies the unit's input (gate and up are linear in it: the factor is applied to their
products, ahead of the clamps).  Logits come from the embedding table, through a soft cap.
"""

from __future__ import annotations

import torch
import torch.nn.functional as F

from .. import ops
from ..engine.config import FeedForwardSpec, LatentMixerSpec, MinGRUSpec, ModelConfig
from ..ops.reference import PAGE
from ..parallel.state import get_pp, get_tp
from .batch import BatchMeta
from .latent_mixer import LatentAttention

GLU_ALPHA = 1.702   # the gated unit: g sigmoid(1.702 g) (u + 1) on clamped g and u
GLU_UP_BIAS = 1.0


class ZupilornLayer:
    __slots__ = ("spec", "norm1", "norm1b", "norm2", "norm2b", "dwa", "w_in", "w_o", "z_bias", "x_bias", "state_off",
                 "dkv_norm", "w_uk", "w_uv", "w_vk", "sink", "cache_offset", "cos_sin", "w_up", "w_down", "act", "router",
                 "w13", "w2")

    def __init__(self, spec):
        for s in self.__slots__:
            setattr(self, s, None)
        self.spec = spec


class ZupilornModel(LatentAttention):
    stateful = True  # sequences carry state slots; a prefix's pages alone do not restore a sequence

    def __init__(self, cfg: ModelConfig, dtype: torch.dtype, device: torch.device, max_model_len: int):
        if get_tp().size != 1 or get_pp().size != 1:
            raise ValueError("Zupilorn runs on single-GPU replicas (no tensor / pipeline parallel layout yet)")
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError("Zupilorn runs in bfloat16 or float32")
        self.cfg = cfg
        self.dtype = dtype
        self.device = device
        self.max_model_len = max_model_len
        self.specs = cfg.layer_specs
        self.n_q = cfg.num_heads
        self.n_kv = 1
        self.head_dim = cfg.head_dim
        self.tp_size = 1
        self.lora = None
        self.layers: list[ZupilornLayer] = []
        self.embed = self.embed_norm = self.norm = None
        self.state: torch.Tensor | None = None  # [slots, state_elems] fp32, bound by the runner
        self.layer_probe = None  # callable(layer index, fp32 residual stream after the layer's average) for tests
        # where each layer's part of a pool page or of a state slot starts, in elements
        self.cache_offsets: dict[int, int] = {}
        self.state_offsets: dict[int, int] = {}
        c_off = s_off = 0
        for i, s in enumerate(self.specs):
            if isinstance(s.mixer, MinGRUSpec):
                self.state_offsets[i] = s_off
                s_off += (s.mixer.state_elems() + 3) // 4 * 4  # parts start on 16-byte boundaries
            else:
                self.cache_offsets[i] = c_off
                c_off += PAGE * s.mixer.entry
        self.page_elems = max(c_off, 8)   # a model of recurrences only still names (empty) pages
        self.state_elems = max(s_off, 8)
        self._tables: dict[tuple, torch.Tensor] = {}

    @property
    def graph_capturable(self) -> bool:
        """Decode steps can be captured when no layer's mixture falls back to the per-unit loop, which reads
        the row counts on the host (shapes the grouped GEMM does not tile, fp32)."""
        probe = torch.empty((1, self.cfg.hidden_size), dtype=self.dtype, device=self.device)
        return self.dtype == torch.bfloat16 and self.device.type == "cuda" and all(
            lw.w13 is None or ops.moe_glu_grouped_supported(probe, lw.w13, lw.w2) for lw in self.layers)

    # ------------------------------------------------------------------ stores
    def kv_page_shape(self) -> tuple:
        """Shape of one page of the KV pool (the runner allocates [pages, *shape])."""
        return (self.page_elems,)

    def state_shape(self) -> tuple:
        """Shape of one sequence's state slot (the runner allocates fp32 [slots, *shape])."""
        return (self.state_elems,)

    def bind_state(self, state: torch.Tensor | None) -> None:
        self.state = state

    # ------------------------------------------------------------------ weights
    def _alloc(self, gen, *shape, std=None, dtype=None, mean=0.0):
        dtype = dtype or self.dtype
        t = torch.empty(shape, dtype=torch.float32, device=self.device)
        t.normal_(mean, std if std is not None else shape[-1] ** -0.5, generator=gen)
        return t.to(dtype)

    def init_random(self, seed: int = 0) -> None:
        """Allocates every tensor in the layout the forward pass uses; a checkpoint overwrites them."""
        cfg = self.cfg
        w = cfg.hidden_size
        g = torch.Generator(device=self.device).manual_seed(seed)
        f32 = torch.float32

        def gain():
            return self._alloc(g, w, std=0.1, dtype=f32, mean=1.0)

        self.embed = self._alloc(g, cfg.vocab_size, w, std=w ** -0.5)
        self.embed_norm = gain()
        self.layers = []
        for i, s in enumerate(self.specs):
            m, f = s.mixer, s.mlp
            lw = ZupilornLayer(s)
            lw.norm1, lw.norm1b = gain(), gain()
            lw.dwa = self._alloc(g, i + 2, std=0.1, dtype=f32)
            lw.dwa[i + 1] += 1.0
            if isinstance(m, MinGRUSpec):
                lw.w_in = self._alloc(g, 3 * m.width, w)
                lw.z_bias = self._alloc(g, m.width, std=1.0, dtype=f32, mean=-2.0)
                lw.x_bias = self._alloc(g, m.width, std=0.3, dtype=f32)
                lw.w_o = self._alloc(g, w, m.width)
                lw.state_off = self.state_offsets[i]
            else:
                lw.w_in = self._alloc(g, m.heads * (m.dim + m.rot_dim) + m.entry, w)
                lw.dkv_norm = self._alloc(g, m.kv_rank, std=0.1, dtype=f32, mean=1.0)
                lw.w_uk = self._alloc(g, m.heads, m.dim, m.kv_rank)
                lw.w_uv = self._alloc(g, m.heads, m.kv_rank, m.vdim, std=m.kv_rank ** -0.5)
                lw.w_o = self._alloc(g, w, m.heads * m.vdim)
                lw.cache_offset = self.cache_offsets[i]
                lw.cos_sin = self._cos_sin(m)
            if f is not None:
                lw.norm2, lw.norm2b = gain(), gain()
                if f.kind == "dense":
                    lw.w_up = self._alloc(g, f.ff, w)
                    lw.w_down = self._alloc(g, w, f.ff)
                    lw.act = self._alloc(g, 4, std=0.5, dtype=f32)
                else:
                    lw.router = self._alloc(g, f.experts, w, dtype=f32)
                    lw.w13 = self._alloc(g, f.experts, 2 * f.ff, w)
                    lw.w2 = self._alloc(g, f.experts, w, f.ff)
            self.layers.append(lw)
        self.norm = gain()

    @property
    def lm_head(self) -> torch.Tensor:  # the embedding table is the output matrix
        return self.embed

    def weight_tensors(self):
        for t in (self.embed, self.embed_norm, self.norm):
            if t is not None:
                yield t
        for lw in self.layers:
            for s in ZupilornLayer.__slots__:
                t = getattr(lw, s)
                if isinstance(t, torch.Tensor) and s not in ("cos_sin", "w_vk"):
                    yield t

    def weight_bytes(self) -> int:
        return sum(t.numel() * t.element_size() for t in self.weight_tensors())

    # ------------------------------------------------------------------ batch description
    def plan_prefill(self, meta: BatchMeta, q_lens: list[int], ctx_lens: list[int], to_dev) -> None:
        mixers = [s.mixer for s in self.specs if isinstance(s.mixer, LatentMixerSpec)]
        if mixers:
            self.plan_latent_prefill(meta, q_lens, ctx_lens, to_dev, mixers)

    def plan_batch(self, meta: BatchMeta, plan: dict, to_dev) -> None:
        """Sequences of the step for the kernels that walk them: decode rows (one row each), then the
        prefill chunks; every sequence with its state slot."""
        q_lens = [1] * plan["num_decode"] + list(plan.get("q_lens", []))
        cu = [0]
        for n in q_lens:
            cu.append(cu[-1] + n)
        meta.seq_cu = to_dev(cu, torch.int32)
        meta.seq_state = to_dev(plan["state_slots"], torch.int32)
        cut = ops.build_gru_pieces(q_lens) if self.device.type == "cuda" else None
        if cut is not None:
            meta.scan_pieces = tuple(torch.from_numpy(a).pin_memory().to(self.device, non_blocking=True) for a in cut)

    def plan_decode_graph(self, meta: BatchMeta, bsz: int, state_slots: torch.Tensor) -> None:
        """The same for a captured decode step of ``bsz`` rows: ``state_slots`` is a graph input."""
        meta.seq_cu = torch.arange(bsz + 1, dtype=torch.int32, device=self.device)
        meta.seq_state = state_slots

    # ------------------------------------------------------------------ sublayers
    def _mingru(self, lw: ZupilornLayer, h: torch.Tensor, meta: BatchMeta) -> torch.Tensor:
        n = lw.spec.mixer.width
        proj = ops.linear(h, lw.w_in)  # z | x | g
        y = ops.mingru_scan(proj, 0, n, 2 * n, n, lw.z_bias, lw.x_bias, self.state, lw.state_off, meta.seq_cu,
                            meta.seq_state, meta.positions, pieces=meta.scan_pieces)
        return ops.linear(y, lw.w_o)

    def _attention(self, lw: ZupilornLayer, h: torch.Tensor, pool, meta: BatchMeta) -> torch.Tensor:
        m: LatentMixerSpec = lw.spec.mixer
        t = h.shape[0]
        nq = m.heads * (m.dim + m.rot_dim)
        proj = ops.linear(h, lw.w_in)  # q | KV latent | shared key part
        q = proj[:, :nq].view(t, m.heads, m.dim + m.rot_dim)
        ops.latent_kv_write(proj[:, nq:nq + m.entry], lw.dkv_norm, meta.positions, meta.slots, lw.cos_sin, pool,
                            lw.cache_offset, m.kv_rank, m.rot_dim, m.rope_dims, self.cfg.norm_eps, q=q, q_col=m.dim)
        o = self.latent_heads(lw, q, pool, meta)
        return ops.linear(o.view(t, m.heads * m.vdim), lw.w_o)

    def _feed_forward(self, lw: ZupilornLayer, h: torch.Tensor) -> torch.Tensor:
        f: FeedForwardSpec = lw.spec.mlp
        if f.kind == "dense":
            return ops.linear(ops.up_poly_norm(h, lw.w_up, lw.act, self.cfg.norm_eps), lw.w_down)
        logits = F.linear(h.float(), lw.router)  # a true fp32 product
        w, ids, _ = ops.group_topk(logits, f.experts, f.groups, f.keep, f.top, f.route_scale)
        ys, pos = ops.moe_glu(h, lw.w13, lw.w2, ids, f.limit, GLU_ALPHA, GLU_UP_BIAS, scale=w)
        if f.top == 1 and ys.dtype == torch.float32:  # nothing to sum
            return ys.index_select(0, pos)
        out = torch.empty(h.shape, dtype=torch.float32, device=h.device)
        return ops.moe_finish(out, ys, None, pos, overwrite=True)

    # ------------------------------------------------------------------ forward
    def forward(self, input_ids: torch.Tensor, pool: torch.Tensor, meta: BatchMeta) -> torch.Tensor:
        """Final-normed hidden states of ``meta.logits_rows`` ([num_out, width], activation dtype)."""
        eps, dt, n = self.cfg.norm_eps, self.dtype, len(self.layers)
        # history[0] the embedding output, history[i + 1] layer i's result (the last one's is not read again)
        history = torch.empty((max(n, 1), input_ids.shape[0], self.cfg.hidden_size), dtype=torch.float32, device=self.device)
        x = ops.embed_rms_norm(input_ids, self.embed, self.embed_norm, eps, out=history[0])
        h = None
        for i, lw in enumerate(self.layers):
            if i == 0:
                h = ops.gated_add_rms_norm(x, [], None, None, lw.norm1, eps, dt)
            d = self._mingru(lw, h, meta) if lw.state_off is not None else self._attention(lw, h, pool, meta)
            after = lw.norm1b
            if lw.spec.mlp is not None:
                h = ops.gated_add_rms_norm(x, [(d, after, 1.0)], None, None, lw.norm2, eps, dt)
                d, after = self._feed_forward(lw, h), lw.norm2b
            last = i + 1 == n
            if last and meta.logits_rows is not None and self.layer_probe is None:
                x, d = x.index_select(0, meta.logits_rows), d.index_select(0, meta.logits_rows)
                history = history.index_select(1, meta.logits_rows)
            h = ops.depth_mix_rms_norm(x, d, after, history, i + 1, not last, lw.dwa,
                                       self.norm if last else self.layers[i + 1].norm1, eps, dt)
            if self.layer_probe is not None:
                self.layer_probe(i, x)
                if last and meta.logits_rows is not None:
                    h = h.index_select(0, meta.logits_rows)
        return h

    def compute_logits(self, hidden: torch.Tensor) -> torch.Tensor:
        logits = ops.linear(hidden, self.embed)
        return ops.soft_cap(logits, self.cfg.logit_softcap) if self.cfg.logit_softcap else logits
