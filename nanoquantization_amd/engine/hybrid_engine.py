"""Paged-KV and recurrent-state execution of HybridDecoder models (models/hybrid.py) on one MI355X.

Residual.  fp32 throughout, and written lazily: what a sublayer leaves is added by the kernel that also computes the next
sublayer's norm.  `Residual` is one row per token; a sublayer may end in a norm of its own, and in front of a repeated pass the
embedding output is added, gathered again from the table instead of being kept.  `Streams` are several rows per token under
hyper-connections.

Caches.  Every layer run (a looped layer runs several times) has its own K/V tensors or its own latent rows, all indexed by
the sequence's one block table, or its own state tensors, indexed by the sequence's state slot.  K/V and latent rows are padded
to a width the matrix-core kernels take.

Latent attention.  Decode steps and short portions take the queries into the latent space and attend to the latents
themselves; longer prompt passes expand the contexts' latents to keys and values per head, which is fewer operations per
query and key.

Entry points.  `extend` runs any number of tokens of any number of sequences from where their caches stand (prompts,
portions of prompts); `_decode_step` runs one token per batch row from the static buffers of EngineCore, in bf16 as a HIP
graph of this library's kernels only.  Both share `_layers`; a `Step` tells the mixers which of the two is running."""
from __future__ import annotations

from dataclasses import dataclass
from typing import Dict, List, Optional, Sequence

import torch
import torch.nn.functional as F

from ..models.hybrid import (AttentionSpec, DenseSpec, GatedLinearSpec, HybridDecoder, LatentAttentionSpec, RotarySpec,
                             SelectiveScanSpec, rotary_table)
from . import hybrid_ops as ops
from .cache import Lease, PagedKVCache, RecurrentStateCache
from .core import EngineCore


@dataclass
class Portion:
    """`tokens` of one sequence at positions start, start + 1, ...; logits are returned for the places in `want`."""
    lease: Lease
    start: int
    tokens: Sequence[int]
    want: Sequence[int]


@dataclass
class Step:
    """The tokens of one pass over the layers: a prompt pass has a layout, a decode step the tokens in each row's cache."""
    ids: torch.Tensor
    positions: torch.Tensor
    slots: torch.Tensor
    layout: Optional[ops.PromptPass] = None
    context: Optional[torch.Tensor] = None


class Residual:
    """One fp32 row per token."""

    def __init__(self, step: Step, table: torch.Tensor, eps: float, width: int):
        self.eps, self.table, self.ids = eps, table, step.ids
        self.x = torch.empty(step.ids.numel(), width, dtype=torch.float32, device=table.device)
        self.pending: dict = dict(init=True, ids=step.ids, table=table)

    def add_embedding(self) -> None:
        self.pending.update(ids=self.ids, table=self.table)

    def read(self, norm: torch.Tensor, hyper=None) -> torch.Tensor:
        return ops.residual_norm(self.x, self.eps, next_weight=norm, **self.pending)

    def read_routed(self, norm: torch.Tensor, router: torch.Tensor, top: int, ff: int):
        return ops.residual_norm_route(self.x, self.eps, router, top, ff, norm, **self.pending)

    def write(self, y: torch.Tensor, post_norm: Optional[torch.Tensor], hyper=None) -> None:
        self.pending = dict(y=y, post_weight=post_norm)

    def select(self, rows: torch.Tensor) -> None:
        """Only these rows go on."""
        self.x = self.x[rows].contiguous()
        if "y" in self.pending:
            self.pending["y"] = self.pending["y"][rows].contiguous()

    def value(self) -> torch.Tensor:
        if self.pending:
            ops.residual_norm(self.x, self.eps, **self.pending)
            self.pending = {}
        return self.x.clone()


class Streams:
    """Several fp32 rows per token; `hyper` is the StreamWeights of the sublayer that reads or writes."""

    def __init__(self, step: Step, table: torch.Tensor, eps: float, width: int, streams: int):
        self.eps = eps
        self.x = torch.empty(step.ids.numel(), streams, width, dtype=torch.float32, device=table.device)
        self.pending: dict = dict(ids=step.ids, table=table)

    def read(self, norm: torch.Tensor, hyper=None) -> torch.Tensor:
        """`hyper` None: the plain sum of the streams."""
        return ops.hyper_norm(self.x, self.eps, read=None if hyper is None else hyper.read, next_weight=norm, **self.pending)

    def write(self, y: torch.Tensor, post_norm: Optional[torch.Tensor], hyper=None) -> None:
        self.pending = dict(y=y, mix=hyper.mix, write=hyper.write)

    def select(self, rows: torch.Tensor) -> None:
        self.x = self.x[rows].contiguous()
        if "y" in self.pending:
            self.pending["y"] = self.pending["y"][rows].contiguous()

    def value(self) -> torch.Tensor:
        if self.pending:
            ops.hyper_norm(self.x, self.eps, **self.pending)
            self.pending = {}
        return self.x.sum(dim=1)


class HybridEngine(EngineCore):
    step_ops = ops
    absorb_rows = ops.SKINNY_ROWS       # prompt passes of up to so many rows attend to latents as a decode step does

    def __init__(self, model: HybridDecoder, max_batch: int, max_seq_len: int, block_size: int = 64,
                 num_blocks: Optional[int] = None, use_graph: bool = True, num_slots: Optional[int] = None,
                 prefill_tokens: int = 8192):
        self.model = model.eval()
        p = model.embed
        self.spec = spec = model.spec
        # a graph may hold this library's kernels only: products in fp32, of odd widths or of many rows are the vendor
        # library's, which may record memory-clearing nodes
        linears = [model.head] + [w for l in model.layers for w in l.linears()]
        super().__init__(p.device, p.dtype, max_batch, max_seq_len, block_size, num_blocks,
                         use_graph and all(ops.skinny_linear_supported(max_batch, w) for w in linears))
        self.runs = spec.runs()
        self.prefill_tokens = prefill_tokens
        mixers = [spec.layers[i].mixer for i, _ in self.runs]
        self.cache = PagedKVCache(len(mixers), self.num_blocks, block_size, dtype=self.dtype, device=self.device,
                                  layer_shapes=[self._cache_shape(m) for m in mixers])
        state_shapes, tail_shapes = zip(*(self._state_shapes(m) for m in mixers))
        if any(state_shapes):
            self.states = RecurrentStateCache(num_slots or max_batch, state_shapes, self.device, tail_shapes)
        self._angles: Dict[RotarySpec, torch.Tensor] = {}
        for rot in (getattr(m, "rotary", None) for m in mixers):
            if rot is not None and rot not in self._angles:
                self._angles[rot] = rotary_table(rot, self.max_ctx).to(self.device)
        # latent attention: the expansions per head, as the products into and out of the latent space want them
        self._per_head = {i: model.layers[i].mixer.per_head() for i, l in enumerate(spec.layers)
                          if isinstance(l.mixer, LatentAttentionSpec)}

    def _cache_shape(self, m):
        if isinstance(m, AttentionSpec):
            return (m.kv_heads, *ops.cache_rows(m.dim, m.vdim, self.dtype))
        if isinstance(m, LatentAttentionSpec):
            return (1, ops.latent_row(m.rank, m.rotary.dims, self.dtype)[1], 0)
        return None

    @staticmethod
    def _state_shapes(m):
        """(recurrent state, last inputs of the convolution) of a run; None: has none."""
        if isinstance(m, GatedLinearSpec):
            return (m.heads, m.dim, m.vdim), None
        if isinstance(m, SelectiveScanSpec):
            return (m.state, m.channels), (m.taps - 1, m.channels)
        return None, None

    # ---- pieces shared by prefill and decode ---------------------------------------------------------
    def _linear(self, x: torch.Tensor, w: torch.Tensor, b: Optional[torch.Tensor] = None, activation: Optional[str] = None,
                param: float = 0.0) -> torch.Tensor:
        if ops.skinny_linear_supported(x.shape[0], w):
            return ops.skinny_linear(x, w, b, activation=activation, param=param)
        y = F.linear(x, w, b)
        return y if activation is None else ops.activate_(y, activation, param)

    def _logits(self, h: torch.Tensor) -> torch.Tensor:
        """fp32 logits of normalised rows."""
        w, cap = self.model.head, self.spec.logit_cap
        act = "softcap" if cap else None
        if h.dtype != torch.float32 and ops.skinny_linear_supported(1, w):
            parts = [ops.skinny_linear(p, w, out_f32=True, activation=act, param=cap) for p in h.split(ops.SKINNY_ROWS)]
            return parts[0] if len(parts) == 1 else torch.cat(parts)
        y = F.linear(h, w).float()
        return ops.activate_(y, act, cap) if act else y

    # ---- mixers: h [rows, width] -> what the output projection takes ------------------------------------
    def _attention(self, run: int, m: AttentionSpec, w, h: torch.Tensor, step: Step) -> torch.Tensor:
        k, v = self.cache.k[run], self.cache.v[run]
        cos_sin = self._angles[m.rotary] if m.rotary is not None else None
        q = ops.qk_norm_rope_store(self._linear(h, w.qkv, w.qkv_bias), w.q_norm, w.k_norm, cos_sin, step.positions, step.slots,
                                   k, v, m.heads, m.dim, m.vdim, self.spec.eps)
        if step.layout is not None:
            return ops.attention_prefill(q, k, v, step.layout, m.dim, m.vdim, m.scale, m.chunk, m.window, w.sink)
        return ops.attention_decode(q, k, v, self.s_table, step.context, m.dim, m.vdim, m.scale, m.chunk, m.window, w.sink)

    def _latent_attention(self, run: int, m: LatentAttentionSpec, w, h: torch.Tensor, step: Step) -> torch.Tensor:
        cache, rot, eps = self.cache.k[run], m.rotary.dims, self.spec.eps
        rot_at, row = ops.latent_row(m.rank, rot, self.dtype)
        proj, cos_sin, rows = self._linear(h, w.proj), self._angles[m.rotary], h.shape[0]
        wide = 0
        if step.layout is not None and rows > self.absorb_rows:
            wide = ops.latent_prefill_query_row(m.dim, rot, m.vdim, m.rank, self.dtype)
        if wide:
            q = ops.latent_store(proj, w.latent_norm, cos_sin, step.positions, step.slots, cache, m.heads, m.dim, rot_at, eps,
                                 wide, m.dim, True)
            latents = ops.latent_gather(cache, step.layout, m.rank, rot, rot_at)
            return ops.latent_attention_prefill(q, F.linear(latents[:, :m.rank], w.expand), latents[:, m.rank:], step.layout,
                                                m.dim, m.vdim, m.scale)
        into, out_of = self._per_head[self.runs[run][0]]
        q = ops.latent_store(proj, w.latent_norm, cos_sin, step.positions, step.slots, cache, m.heads, m.dim, rot_at, eps, row,
                             rot_at, False)
        ops.head_linear(proj[:, :w.splits[0]].view(rows, m.heads, m.dim + rot), into, q)
        if step.layout is None:
            o = ops.latent_attention_decode(q, cache, self.s_table, step.context, m.rank, rot_at, m.scale)
        elif rows <= self.absorb_rows:
            o = ops.latent_attention_decode(q, cache, *step.layout.row_tables(), m.rank, rot_at, m.scale)
        else:       # the latent row as key and as value of a single head
            o = ops.attention_prefill(q, cache, cache, step.layout, row, m.rank, m.scale).view(rows, m.heads, m.rank)
        return ops.head_linear(o, out_of, torch.empty(rows, m.heads, m.vdim, dtype=o.dtype, device=o.device)).view(rows, -1)

    def _gated_linear(self, run: int, m: GatedLinearSpec, w, h: torch.Tensor, step: Step) -> torch.Tensor:
        proj, state = self._linear(h, w.proj), self.states.state[run]
        if step.layout is None:
            return ops.gla_decode(proj, w.decay_up, w.decay_bias, w.head_norm, state, self.s_slot, self.s_pos, self.s_active,
                                  m.heads, m.dim, m.vdim, m.tau, self.spec.eps)
        decay = ops.gla_decay(proj, w.decay_up, w.decay_bias, m.heads, m.dim, m.vdim, m.tau)
        o = ops.gla_prefill(proj, decay, state, step.layout, m.heads, m.dim, m.vdim, m.rank)
        return ops.head_norm_gate(o, proj, w.head_norm, m.heads, m.dim, m.vdim, m.rank, self.spec.eps)

    def _selective_scan(self, run: int, m: SelectiveScanSpec, w, h: torch.Tensor, step: Step) -> torch.Tensor:
        state, tail = self.states.state[run], self.states.tail[run]
        x_in, z = self._linear(h, w.proj).split([m.channels, m.channels], dim=1)
        if step.layout is None:
            x = ops.conv_step(x_in, w.conv, w.conv_bias, tail, self.s_slot, self.s_pos, self.s_active)
        else:
            piece = ops.scan_piece_rows(h.shape[0], m.channels, m.state)
            x = ops.conv_silu(x_in, w.conv, w.conv_bias, tail, step.layout, piece)
        low, bc = self._linear(x, w.select).split([m.dt_rank, 2 * m.state], dim=1)
        dt = ops.scan_dt(low, w.dt_up, w.dt_bias)
        if step.layout is None:
            return ops.scan_step(x, dt, bc, z, w.a_log, w.skip, state, self.s_slot, self.s_pos, self.s_active)
        return ops.scan_prefill(x, dt, bc, z, w.a_log, w.skip, x_in, state, tail, step.layout, piece)

    _MIXERS = {AttentionSpec: _attention, LatentAttentionSpec: _latent_attention, GatedLinearSpec: _gated_linear,
               SelectiveScanSpec: _selective_scan}

    def _layers(self, step: Step, rows: Optional[torch.Tensor] = None, trace: Optional[list] = None) -> torch.Tensor:
        """All layer runs for the given tokens; returns the final norm of the residual rows `rows` (all if None).  `trace`
        receives the residual (the sum of its streams) after every run (costs extra launches)."""
        model, spec = self.model, self.spec
        args = (step, model.embed, spec.eps, spec.width)
        res = Streams(*args, spec.streams) if spec.streams else Residual(*args)
        for run, (li, add_embedding) in enumerate(self.runs):
            layer, ls = model.layers[li], spec.layers[li]
            if add_embedding:
                res.add_embedding()
            h = res.read(layer.norm_mixer, layer.mixer_streams)
            o = self._MIXERS[type(ls.mixer)](self, run, ls.mixer, layer.mixer, h, step)
            res.write(self._linear(o, layer.mixer.out), layer.norm_mixer_out, layer.mixer_streams)
            if isinstance(ls.mlp, DenseSpec):
                h = res.read(layer.norm_mlp, layer.mlp_streams)
                y = self._linear(self._linear(h, layer.mlp.up, activation=ls.mlp.activation), layer.mlp.down)
                res.write(y, layer.norm_mlp_out, layer.mlp_streams)
            elif ls.mlp is not None:
                h, routing = res.read_routed(layer.norm_mlp, layer.mlp.router, ls.mlp.top, ls.mlp.ff)
                res.write(ops.moe_experts(h, layer.mlp.gate_up, layer.mlp.down, routing), layer.norm_mlp_out)
            if trace is not None:
                trace.append(res.value())
        if rows is not None:
            res.select(rows)
        return res.read(model.final_norm)

    # ---- any number of tokens of any number of sequences ------------------------------------------------
    @torch.no_grad()
    def extend(self, portions: List[Portion], trace: Optional[list] = None) -> torch.Tensor:
        """Run the portions from the cache and state their sequences have; one pass.  Returns fp32 logits, one row per
        wanted place in order."""
        bs, dev = self.block_size, self.device
        ids, pos, slots, want, first = [], [], [], [], 0
        for p in portions:
            n = len(p.tokens)
            if n < 1 or p.start < 0 or p.start + n > min(len(p.lease.blocks) * bs, self.max_ctx):
                raise ValueError(f"{n} tokens from position {p.start} do not fit the sequence's "
                                 f"{len(p.lease.blocks)} blocks of {bs} tokens")
            if min(p.tokens) < 0 or max(p.tokens) >= self.spec.vocab:
                raise ValueError("token id outside the vocabulary")
            ids += p.tokens
            t = range(p.start, p.start + n)
            pos += t
            slots += [p.lease.blocks[i // bs] * bs + i % bs for i in t]
            want += [first + w for w in p.want]
            first += n
        layout = ops.PromptPass([(p.start, len(p.tokens), p.lease.blocks, p.lease.slot) for p in portions], bs, dev)
        packed = torch.tensor([ids, pos, slots], dtype=torch.long).to(dev)
        ids_d, pos_d, slots_d = packed[0], packed[1], packed[2]

        step = Step(ids_d, pos_d, slots_d, layout=layout)
        rows = torch.tensor(want, dtype=torch.long).to(dev)
        if not want:        # the pass still fills cache and state
            self._layers(step, trace=trace)
            return torch.empty(0, self.spec.vocab, dtype=torch.float32, device=dev)
        return self._logits(self._layers(step, rows, trace))

    def _prefill_ragged(self, prompts: List[List[int]], leases: List[Lease]) -> torch.Tensor:
        """Whole prompts; longer ones than `prefill_tokens` in portions, the rest of the pass filled with the next."""
        out: List[Optional[torch.Tensor]] = [None] * len(prompts)
        batch: List[Portion] = []
        owners: List[int] = []
        room = self.prefill_tokens

        def flush():
            nonlocal room
            if batch:
                logits = self.extend(batch)
                if owners:
                    for i, tok in zip(owners, ops.argmax_rows(logits)):
                        out[i] = tok
            batch.clear(); owners.clear()
            room = self.prefill_tokens
        for i, (prompt, lease) in enumerate(zip(prompts, leases)):
            at = 0
            while at < len(prompt):
                n = min(room, len(prompt) - at)
                last = at + n == len(prompt)
                batch.append(Portion(lease, at, prompt[at:at + n], [n - 1] if last else []))
                if last:
                    owners.append(i)
                at, room = at + n, room - n
                if room == 0:
                    flush()
        flush()
        return torch.stack(out)

    def _prefill(self, ids: torch.Tensor, leases: List[Lease]) -> torch.Tensor:
        return self._prefill_ragged(ids.tolist(), leases)

    # ---- one token per batch row -----------------------------------------------------------------------
    def _decode_step(self) -> None:
        slots, ctx = ops.decode_prepare(self.s_pos, self.s_active, self.s_table, self.block_size)
        self._finish_step(self._logits(self._layers(Step(self.s_ids, self.s_pos, slots, context=ctx))))
