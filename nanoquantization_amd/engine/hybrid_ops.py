"""torch-tensor wrappers of the kernels declared in include/nq_hybrid_ops.h.

Each function checks shapes on the host, allocates its output with torch (graph-capture safe: the caching allocator)
and launches on the current stream.  HIP device tensors only; bfloat16 or float32."""
from __future__ import annotations

from typing import Optional, Sequence, Tuple

import torch

from .. import _lib

_DTYPES = {torch.bfloat16: 1, torch.float32: 2}
SKINNY_ROWS = 64
ACTIVATIONS = {None: 0, "relu2": 1, "softcap": 2}      # what may follow a product; "softcap" takes the cap as parameter

_MATRIX_ROWS = (32, 64, 96, 128, 192, 256)      # cache row widths the matrix-core attention kernels exist for


def cache_rows(dim: int, vdim: int, dtype: torch.dtype) -> Tuple[int, int]:
    """Width of a K and of a V cache row for heads of `dim` and `vdim` elements: in bf16 the smallest width the
    matrix-core kernels take for both, in fp32 the heads as they are."""
    if dtype == torch.float32:
        return dim, vdim
    for row in _MATRIX_ROWS:
        if max(dim, vdim) <= row:
            return row, row
    return (dim + 31) // 32 * 32, (vdim + 31) // 32 * 32


def latent_row(rank: int, rot_dim: int, dtype: torch.dtype) -> Tuple[int, int]:
    """(place of the rotated part, width) of a latent cache row: in bf16 padded to what the matrix-core kernel takes, in
    fp32 and beyond its sizes without padding."""
    if dtype == torch.bfloat16 and rank <= 512 and rot_dim <= 64:
        at = next(r for r in (64, 128, 256, 512) if rank <= r)
        return at, at + (32 if rot_dim <= 32 else 64)
    return rank, rank + rot_dim


def _dtype(t: torch.Tensor) -> int:
    if t.dtype not in _DTYPES:
        raise _lib.AwqHipError(f"hybrid kernels take bfloat16 or float32, got {t.dtype}")
    return _DTYPES[t.dtype]


def _dev(*ts: Optional[torch.Tensor]) -> torch.device:
    dev = ts[0].device
    if dev.type != "cuda":
        raise _lib.AwqHipError(f"engine kernels run on a HIP device only (tensor is on {dev})")
    for t in ts:
        if t is not None and t.device != dev:
            raise _lib.AwqHipError(f"tensors on different devices: {t.device} vs {dev}")
        if t is not None and not t.is_contiguous():
            raise _lib.AwqHipError("engine kernels take contiguous tensors")
    return dev


def _ptr(t: Optional[torch.Tensor]):
    return None if t is None else t.data_ptr()


def _call(dev: torch.device, fn: str, *args) -> None:
    with _lib.on_device(dev):
        _lib.check_hybrid(getattr(_lib.hybrid_lib(), fn)(*args, _lib.current_stream_ptr(dev)))


def _residual_args(x, eps, y, post_weight, ids, table, init, next_weight, dtype):
    dev = _dev(x, y, post_weight, ids, table, next_weight)
    rows, width = x.shape
    assert x.dtype == torch.float32
    operands = [t for t in (y, post_weight, table, next_weight) if t is not None]
    dt = operands[0].dtype if operands else dtype
    assert all(t.dtype == dt for t in operands)
    parts = 1
    if y is not None:
        parts = 1 if y.dim() == 2 else y.shape[1]
        assert y.shape[0] == rows and y.shape[-1] == width
    assert post_weight is None or post_weight.shape == (width,)
    assert next_weight is None or next_weight.shape == (width,)
    if ids is not None:
        assert ids.dtype == torch.int64 and ids.numel() == rows and table.shape[1] == width
    h = torch.empty(rows, width, dtype=dt, device=dev) if next_weight is not None else None
    return dev, h, dt, (x.data_ptr(), int(init), _ptr(y), parts, _ptr(post_weight), _ptr(ids), _ptr(table),
                        0 if table is None else table.shape[0], _ptr(next_weight), _ptr(h))


def residual_norm(x: torch.Tensor, eps: float, *, y: Optional[torch.Tensor] = None, post_weight: Optional[torch.Tensor] = None,
                  ids: Optional[torch.Tensor] = None, table: Optional[torch.Tensor] = None, init: bool = False,
                  next_weight: Optional[torch.Tensor] = None, dtype: Optional[torch.dtype] = None) -> Optional[torch.Tensor]:
    """The fp32 residual stream x [rows, width] IN PLACE: (0 if init) + RMSNorm(sum over parts of y [rows, parts, width]) *
    post_weight + table[ids]; returns RMSNorm(x) * next_weight (None without next_weight)."""
    dev, h, dt, args = _residual_args(x, eps, y, post_weight, ids, table, init, next_weight, dtype)
    _call(dev, "nqh_residual_norm", *args, *x.shape, eps, _DTYPES[dt])
    return h


def hyper_norm(x: torch.Tensor, eps: float, *, ids: Optional[torch.Tensor] = None, table: Optional[torch.Tensor] = None,
               y: Optional[torch.Tensor] = None, mix: Optional[torch.Tensor] = None, write: Optional[torch.Tensor] = None,
               read: Optional[torch.Tensor] = None, next_weight: Optional[torch.Tensor] = None) -> Optional[torch.Tensor]:
    """The fp32 residual streams x [rows, streams, width] IN PLACE: all set to table[ids], or mixed anew from the old ones
    and a sublayer's output y; returns RMSNorm(sum of the streams times read, or of the streams as they are) * next_weight
    (None without next_weight)."""
    dev = _dev(x, ids, table, y, mix, write, read, next_weight)
    rows, streams, width = x.shape
    assert x.dtype == torch.float32
    operands = [t for t in (table, y, mix, write, read, next_weight) if t is not None]
    dt = operands[0].dtype
    assert all(t.dtype == dt for t in operands)
    assert ids is None or (y is None and ids.dtype == torch.int64 and ids.numel() == rows and table.shape[1] == width)
    assert y is None or (y.shape == (rows, width) and mix.shape == (streams, streams) and write.shape == (streams,))
    assert read is None or read.shape == (streams,)
    assert next_weight is None or next_weight.shape == (width,)
    h = torch.empty(rows, width, dtype=dt, device=dev) if next_weight is not None else None
    _call(dev, "nqh_hyper_norm", x.data_ptr(), _ptr(ids), _ptr(table), 0 if table is None else table.shape[0], _ptr(y),
          _ptr(mix), _ptr(write), _ptr(read), _ptr(next_weight), _ptr(h), rows, streams, width, eps, _DTYPES[dt])
    return h


def activate_(x: torch.Tensor, activation: str, param: float = 0.0) -> torch.Tensor:
    """activation(x) IN PLACE."""
    _call(_dev(x), "nqh_activate", x.data_ptr(), x.numel(), ACTIVATIONS[activation], param, _dtype(x))
    return x


class Routing:
    """Experts and scores of every row ([rows, top] int32 / fp32) and the grouping of the (row, choice) pairs by expert."""

    def __init__(self, rows: int, experts: int, top: int, width: int, ff: int, dtype: int, dev: torch.device):
        L = _lib.hybrid_lib()
        self.pairs, self.experts, self.top = rows * top, experts, top
        self.tile_rows = L.nqh_moe_tile_rows(self.pairs, experts, width, ff, dtype)
        self.max_tiles = L.nqh_moe_max_tiles(self.pairs, experts, self.tile_rows)
        self.expert = torch.empty(rows, top, dtype=torch.int32, device=dev)
        self.weight = torch.empty(rows, top, dtype=torch.float32, device=dev)
        self.order = torch.empty(self.pairs, dtype=torch.int32, device=dev)
        self.tiles = torch.empty(3 * self.max_tiles + 1, dtype=torch.int32, device=dev)


def residual_norm_route(x: torch.Tensor, eps: float, router: torch.Tensor, top: int, ff: int, next_weight: torch.Tensor, *,
                        y: Optional[torch.Tensor] = None, post_weight: Optional[torch.Tensor] = None,
                        ids: Optional[torch.Tensor] = None, table: Optional[torch.Tensor] = None,
                        init: bool = False) -> Tuple[torch.Tensor, Routing]:
    """residual_norm, the router on its result and the plan of the experts: (h, Routing).  One launch for few rows, three
    otherwise."""
    rows, width = x.shape
    experts = router.shape[0]
    assert router.shape == (experts, width) and router.dtype == next_weight.dtype
    if not _lib.hybrid_lib().nqh_residual_norm_route_supported(rows, width, experts):
        h = residual_norm(x, eps, y=y, post_weight=post_weight, ids=ids, table=table, init=init, next_weight=next_weight)
        return h, route(h, router, top, ff)
    dev, h, dt, args = _residual_args(x, eps, y, post_weight, ids, table, init, next_weight, None)
    _dev(router)
    r = Routing(rows, experts, top, width, ff, _DTYPES[dt], dev)
    counter = _lib.workspace(dev, _lib.current_stream_ptr(dev), 4)       # zero between launches; see _lib.workspace
    _call(dev, "nqh_residual_norm_route", *args, router.data_ptr(), r.expert.data_ptr(), r.weight.data_ptr(),
          r.order.data_ptr(), r.tiles.data_ptr(), counter.data_ptr(), rows, width, experts, top, r.tile_rows, r.max_tiles,
          eps, _DTYPES[dt])
    return h, r


def qk_norm_rope_store(qkv: torch.Tensor, q_weight: Optional[torch.Tensor], k_weight: Optional[torch.Tensor],
                       cos_sin: Optional[torch.Tensor], positions: torch.Tensor, slots: torch.Tensor, k_cache: torch.Tensor,
                       v_cache: torch.Tensor, heads: int, dim: int, vdim: int, eps: float) -> torch.Tensor:
    """qkv [rows, heads * dim + kv_heads * (dim + vdim)]: norm over the whole q and k projections, interleaved rotary on
    the first cos_sin.shape[1] dims of every head, k and v into their cache rows [blocks, kv_heads, block_size, row].
    Returns q [rows, heads, k row]."""
    dev = _dev(qkv, q_weight, k_weight, cos_sin, positions, slots, k_cache, v_cache)
    rows = qkv.shape[0]
    blocks, kv_heads, block_size, k_row = k_cache.shape
    v_row = v_cache.shape[3]
    assert v_cache.shape[:3] == k_cache.shape[:3] and k_cache.dtype == qkv.dtype and v_cache.dtype == qkv.dtype
    assert qkv.shape[1] == heads * dim + kv_heads * (dim + vdim)
    assert (q_weight is None) == (k_weight is None)
    if q_weight is not None:
        assert q_weight.shape == (heads * dim,) and k_weight.shape == (kv_heads * dim,)
        assert q_weight.dtype == qkv.dtype and k_weight.dtype == qkv.dtype
    rot = 0 if cos_sin is None else cos_sin.shape[1]
    assert cos_sin is None or cos_sin.dtype == torch.float32
    assert positions.dtype == torch.int64 and slots.dtype == torch.int64
    assert positions.numel() == rows and slots.numel() == rows
    q = torch.empty(rows, heads, k_row, dtype=qkv.dtype, device=dev)
    _call(dev, "nqh_qk_norm_rope_store", qkv.data_ptr(), _ptr(q_weight), _ptr(k_weight), _ptr(cos_sin),
          positions.data_ptr(), slots.data_ptr(), q.data_ptr(), k_cache.data_ptr(), v_cache.data_ptr(), rows, heads,
          kv_heads, dim, vdim, rot, k_row, v_row, 1 if cos_sin is None else cos_sin.shape[0], blocks * block_size,
          block_size, eps, _dtype(qkv))
    return q


def _check_attention(q, k_cache, v_cache, heads):
    blocks, kv_heads, block_size, k_row = k_cache.shape
    assert v_cache.shape[:3] == k_cache.shape[:3] and k_cache.dtype == q.dtype and v_cache.dtype == q.dtype
    assert q.shape[1:] == (heads, k_row)
    return blocks, kv_heads, block_size, k_row, v_cache.shape[3]


class PromptPass:
    """The layout of a pass over portions of several sequences: segment i is `rows` consecutive tokens of one sequence from
    position `start`, with the cache blocks `blocks` and the state slot `slot`; the segments' tokens lie one after the
    other.  Holds the device-side lists of the prompt kernels."""

    def __init__(self, segments: Sequence[Tuple[int, int, Sequence[int], int]], block_size: int, device: torch.device):
        self.segments = list(segments)                       # (start, rows, blocks, slot)
        self.device = device
        self.rows = sum(s[1] for s in self.segments)
        tile = _lib.hybrid_lib().nqh_attention_tile_rows()
        width = max(1, max(len(s[2]) for s in self.segments))
        table, seg, tiles, first = [], [], [], 0
        for i, (start, rows, blocks, _) in enumerate(self.segments):
            if rows < 1 or start < 0 or start + rows > len(blocks) * block_size:
                raise _lib.AwqHipError(f"segment {i}: positions {start} to {start + rows - 1} do not fit {len(blocks)} blocks")
            table += list(blocks) + [0] * (width - len(blocks))
            seg += [first, rows, start]
            tiles += [(min(start + q0 + tile, start + rows), i, q0) for q0 in range(0, rows, tile)]
            first += rows
        tiles.sort(reverse=True)                             # the tiles with the most keys first
        flat = [x for _, i, q0 in tiles for x in (i, q0)]
        self.num_tiles, self.max_blocks = len(tiles), width
        packed = torch.tensor(table + seg + flat, dtype=torch.int32).to(device)
        self.tables, self.seg, self.tiles = packed.split([len(table), len(seg), len(flat)])
        self._pieces, self._contexts, self._row_tables = {}, None, None

    def contexts(self) -> Tuple[torch.Tensor, int, int]:
        """The segments' contexts laid out one after the other: (first row of each, int32; rows in all; the longest)."""
        if self._contexts is None:
            lens = [start + rows for start, rows, _, _ in self.segments]
            first = [sum(lens[:i]) for i in range(len(lens))]
            self._contexts = torch.tensor(first, dtype=torch.int32).to(self.device), sum(lens), max(lens)
        return self._contexts

    def row_tables(self) -> Tuple[torch.Tensor, torch.Tensor]:
        """The pass as a decode step sees it, every token a row of its own: (block tables [rows, max_blocks], tokens in the
        cache up to and including it [rows])."""
        if self._row_tables is None:
            seg = [i for i, s in enumerate(self.segments) for _ in range(s[1])]
            ctx = [s[0] + t + 1 for s in self.segments for t in range(s[1])]
            seg, ctx = torch.tensor([seg, ctx], dtype=torch.int32).to(self.device)
            self._row_tables = self.tables.view(len(self.segments), self.max_blocks)[seg.long()].contiguous(), ctx.contiguous()
        return self._row_tables

    def pieces(self, size: int) -> Tuple[torch.Tensor, int, bool]:
        """(list of pieces of at most `size` rows for gla_prefill and scan_prefill, its length, whether a sequence has
        several)."""
        if size not in self._pieces:
            out, first, chained = [], 0, False
            for start, rows, _, slot in self.segments:
                n = (rows + size - 1) // size
                chained |= n > 1
                for p in range(n):
                    out += [first + p * size, min(size, rows - p * size), slot, int(start == 0), p, n]
                first += rows
            self._pieces[size] = torch.tensor(out, dtype=torch.int32).to(self.device), len(out) // 6, chained
        return self._pieces[size]


def attention_prefill(q: torch.Tensor, k_cache: torch.Tensor, v_cache: torch.Tensor, layout: PromptPass, dim: int, vdim: int,
                      scale: float, chunk: int = 0, window: int = 0, sink: Optional[torch.Tensor] = None) -> torch.Tensor:
    """q [rows, heads, k row]: the tokens of the pass, attending to their sequences' caches (their own keys are already
    there).  chunk > 0: only keys of the query's own chunk of that many positions; window > 0: only the query's own and the
    window - 1 positions before it.  sink [heads]: a further unscaled score per head, without key or value.  Returns
    [rows, heads * vdim]."""
    rows, heads = q.shape[:2]
    dev = _dev(q, k_cache, v_cache, sink, layout.tables)
    assert sink is None or (sink.shape == (heads,) and sink.dtype == q.dtype)
    blocks, kv_heads, block_size, k_row, v_row = _check_attention(q, k_cache, v_cache, heads)
    assert rows == layout.rows
    out = torch.empty(rows, heads * vdim, dtype=q.dtype, device=dev)
    _call(dev, "nqh_attention_prefill", q.data_ptr(), k_cache.data_ptr(), v_cache.data_ptr(), layout.tables.data_ptr(),
          layout.seg.data_ptr(), layout.tiles.data_ptr(), _ptr(sink), out.data_ptr(), rows, layout.num_tiles, heads, kv_heads,
          dim, vdim, k_row, v_row, block_size, layout.max_blocks, blocks, chunk, window, scale, _dtype(q))
    return out


def attention_decode(q: torch.Tensor, k_cache: torch.Tensor, v_cache: torch.Tensor, block_table: torch.Tensor,
                     context_lens: torch.Tensor, dim: int, vdim: int, scale: float, chunk: int = 0, window: int = 0,
                     sink: Optional[torch.Tensor] = None) -> torch.Tensor:
    """One query token per sequence, the last of its context_lens [batch] int32 cached tokens; block_table int32
    [batch, max_blocks].  Returns [batch, heads * vdim]."""
    batch, heads = q.shape[:2]
    dev = _dev(q, k_cache, v_cache, block_table, context_lens, sink)
    assert sink is None or (sink.shape == (heads,) and sink.dtype == q.dtype)
    blocks, kv_heads, block_size, k_row, v_row = _check_attention(q, k_cache, v_cache, heads)
    assert block_table.dtype == torch.int32 and block_table.dim() == 2 and block_table.shape[0] == batch
    assert context_lens.dtype == torch.int32 and context_lens.shape == (batch,)
    max_blocks = block_table.shape[1]
    out = torch.empty(batch, heads * vdim, dtype=q.dtype, device=dev)
    nbytes = _lib.hybrid_lib().nqh_attention_decode_workspace_bytes(batch, heads, kv_heads, v_row, block_size * max_blocks,
                                                                    chunk, window, _dtype(q))
    ws = torch.empty(nbytes, dtype=torch.uint8, device=dev) if nbytes else None
    _call(dev, "nqh_attention_decode", q.data_ptr(), k_cache.data_ptr(), v_cache.data_ptr(), block_table.data_ptr(),
          context_lens.data_ptr(), _ptr(sink), out.data_ptr(), batch, heads, kv_heads, dim, vdim, k_row, v_row, block_size,
          max_blocks, blocks, chunk, window, scale, _dtype(q), _ptr(ws), nbytes)
    return out


# ---- latent attention --------------------------------------------------------------------------------------------------
def latent_store(proj: torch.Tensor, norm_weight: torch.Tensor, cos_sin: torch.Tensor, positions: torch.Tensor,
                 slots: torch.Tensor, cache: torch.Tensor, heads: int, dim: int, rot_at: int, eps: float, q_row: int,
                 rot_q: int, copy_plain: bool) -> torch.Tensor:
    """proj [rows, heads * (dim + rot) + rank + rot]: the latent normalised and the shared key part rotated into their cache
    rows [blocks, 1, block_size, row]; returns q [rows, heads, q_row] with the rotated part at rot_q and, if copy_plain, the
    unrotated one in front (else that place is left to head_linear)."""
    dev = _dev(proj, norm_weight, cos_sin, positions, slots, cache)
    rows, rot_dim, rank = proj.shape[0], cos_sin.shape[1], norm_weight.shape[0]
    blocks, one, block_size, row = cache.shape
    assert one == 1 and proj.shape[1] == heads * (dim + rot_dim) + rank + rot_dim
    assert norm_weight.dtype == proj.dtype and cache.dtype == proj.dtype and cos_sin.dtype == torch.float32
    assert positions.dtype == torch.int64 and slots.dtype == torch.int64
    assert positions.numel() == rows and slots.numel() == rows
    q = torch.empty(rows, heads, q_row, dtype=proj.dtype, device=dev)
    _call(dev, "nqh_latent_store", proj.data_ptr(), norm_weight.data_ptr(), cos_sin.data_ptr(), positions.data_ptr(),
          slots.data_ptr(), q.data_ptr(), cache.data_ptr(), rows, heads, dim, rot_dim, rank, q_row, rot_q, int(copy_plain),
          row, rot_at, cos_sin.shape[0], blocks * block_size, eps, _dtype(proj))
    return q


def head_linear(x: torch.Tensor, weight: torch.Tensor, y: torch.Tensor) -> torch.Tensor:
    """y[r, h, :out] = weight[h] x[r, h, :in] for weight [heads, out, in]; x and y are 3-d, last dimension dense, and may be
    views."""
    heads, n_out, n_in = weight.shape
    dev = _dev(weight)
    assert x.device == dev and y.device == dev and x.dtype == weight.dtype and y.dtype == weight.dtype
    rows = x.shape[0]
    assert x.shape[1] == heads and x.shape[2] >= n_in and y.shape[:2] == (rows, heads) and y.shape[2] >= n_out
    assert x.stride(2) == 1 and y.stride(2) == 1
    _call(dev, "nqh_head_linear", x.data_ptr(), weight.data_ptr(), y.data_ptr(), rows, heads, n_out, n_in, x.stride(0),
          x.stride(1), y.stride(0), y.stride(1), _dtype(weight))
    return y


def latent_prefill_query_row(dim: int, rot_dim: int, vdim: int, rank: int, dtype: torch.dtype) -> int:
    """Width of a query row for latent_attention_prefill; 0 if it does not take these sizes."""
    if dtype not in _DTYPES or rank % 8:
        return 0
    return _lib.hybrid_lib().nqh_latent_attention_prefill_query_row(dim, rot_dim, vdim, _DTYPES[dtype])


def latent_gather(cache: torch.Tensor, layout: PromptPass, rank: int, rot_dim: int, rot_at: int) -> torch.Tensor:
    """[rows of all contexts, rank + rot_dim]: the cached rows of the segments' contexts without their padding."""
    dev = _dev(cache, layout.tables)
    first, total, longest = layout.contexts()
    blocks, _, block_size, row = cache.shape
    assert cache.element_size() == 2
    out = torch.empty(total, rank + rot_dim, dtype=cache.dtype, device=dev)
    _call(dev, "nqh_latent_gather", cache.data_ptr(), layout.tables.data_ptr(), layout.seg.data_ptr(), first.data_ptr(),
          out.data_ptr(), len(layout.segments), longest, rank, rot_dim, row, rot_at, block_size, layout.max_blocks, blocks)
    return out


def latent_attention_prefill(q: torch.Tensor, kv: torch.Tensor, rot: torch.Tensor, layout: PromptPass, dim: int, vdim: int,
                             scale: float) -> torch.Tensor:
    """q [rows, heads, latent_prefill_query_row]; kv [context rows, heads * (dim + vdim)] and rot [context rows, rot] (a view
    with dense rows is enough) of the contexts as `latent_gather` lays them out.  Returns [rows, heads * vdim]."""
    dev = _dev(q, layout.tables)
    rows, heads = q.shape[:2]
    first, total, _ = layout.contexts()
    assert rows == layout.rows and kv.shape == (total, heads * (dim + vdim)) and rot.shape[0] == total
    assert kv.dtype == q.dtype == rot.dtype == torch.bfloat16 and kv.stride(1) == 1 and rot.stride(1) == 1
    assert q.shape[2] == _lib.hybrid_lib().nqh_latent_attention_prefill_query_row(dim, rot.shape[1], vdim, _dtype(q))
    out = torch.empty(rows, heads * vdim, dtype=q.dtype, device=dev)
    _call(dev, "nqh_latent_attention_prefill", q.data_ptr(), kv.data_ptr(), kv.stride(0), rot.data_ptr(), rot.stride(0),
          first.data_ptr(), layout.seg.data_ptr(), layout.tiles.data_ptr(), out.data_ptr(), rows, layout.num_tiles, heads,
          dim, rot.shape[1], vdim, scale)
    return out


def latent_attention_decode(q: torch.Tensor, cache: torch.Tensor, block_table: torch.Tensor, context_lens: torch.Tensor,
                            rank: int, rot_at: int, scale: float) -> torch.Tensor:
    """One query token per row, q [batch, heads, row] in the latent space; returns [batch, heads, rank] in it."""
    dev = _dev(q, cache, block_table, context_lens)
    batch, heads, row = q.shape
    blocks, one, block_size, width = cache.shape
    assert one == 1 and width == row and cache.dtype == q.dtype
    assert block_table.dtype == torch.int32 and block_table.dim() == 2 and block_table.shape[0] == batch
    assert context_lens.dtype == torch.int32 and context_lens.shape == (batch,)
    max_blocks = block_table.shape[1]
    out = torch.empty(batch, heads, rank, dtype=q.dtype, device=dev)
    nbytes = _lib.hybrid_lib().nqh_latent_attention_decode_workspace_bytes(batch, heads, rank, rot_at, row,
                                                                           block_size * max_blocks, _dtype(q))
    ws = torch.empty(nbytes, dtype=torch.uint8, device=dev) if nbytes else None
    _call(dev, "nqh_latent_attention_decode", q.data_ptr(), cache.data_ptr(), block_table.data_ptr(), context_lens.data_ptr(),
          out.data_ptr(), batch, heads, rank, rot_at, row, block_size, max_blocks, blocks, scale, _dtype(q), _ptr(ws), nbytes)
    return out


# ---- selective scan ------------------------------------------------------------------------------------------------------
def scan_piece_rows(rows: int, channels: int, states: int) -> int:
    return _lib.hybrid_lib().nqh_scan_piece_rows(rows, channels, states)


def _rows_of(t: torch.Tensor, dev: torch.device, width: int) -> None:
    """t is a view of `width` columns with dense rows."""
    assert t.device == dev and t.dim() == 2 and t.shape[1] == width and t.stride(1) == 1


def conv_silu(x: torch.Tensor, weight: torch.Tensor, bias: torch.Tensor, tail: torch.Tensor, layout: PromptPass,
              piece_rows: int) -> torch.Tensor:
    """silu(causal convolution per channel + bias) of the pass's rows x [rows, channels] (a view); `tail` [slots, taps - 1,
    channels] supplies the inputs ahead of a portion and is left as it is (scan_prefill moves it on)."""
    dev = _dev(weight, bias, tail, layout.tables)
    channels, taps = weight.shape
    _rows_of(x, dev, channels)
    assert x.shape[0] == layout.rows and bias.shape == (channels,) and weight.dtype == bias.dtype == x.dtype
    assert tail.dtype == torch.float32 and tail.shape[1:] == (taps - 1, channels)
    assert all(0 <= s[3] < tail.shape[0] for s in layout.segments)
    pieces, n, _ = layout.pieces(piece_rows)
    out = torch.empty(layout.rows, channels, dtype=x.dtype, device=dev)
    _call(dev, "nqh_conv_silu", x.data_ptr(), x.stride(0), weight.data_ptr(), bias.data_ptr(), tail.data_ptr() or None,
          pieces.data_ptr(), n, min(piece_rows, max(s[1] for s in layout.segments)), out.data_ptr(), channels, taps, _dtype(x))
    return out


def conv_step(x: torch.Tensor, weight: torch.Tensor, bias: torch.Tensor, tail: torch.Tensor, slots: torch.Tensor,
              positions: torch.Tensor, active: torch.Tensor) -> torch.Tensor:
    """The same for one token per sequence; `tail` is moved on IN PLACE at the rows' slots."""
    dev = _dev(weight, bias, tail, slots, positions, active)
    channels, taps = weight.shape
    _rows_of(x, dev, channels)
    batch = x.shape[0]
    assert bias.shape == (channels,) and weight.dtype == bias.dtype == x.dtype
    assert tail.dtype == torch.float32 and tail.shape[1:] == (taps - 1, channels)
    assert slots.dtype == torch.int32 and positions.dtype == torch.int64 and active.dtype == torch.bool
    assert slots.numel() == batch and positions.numel() == batch and active.numel() == batch
    out = torch.empty(batch, channels, dtype=x.dtype, device=dev)
    _call(dev, "nqh_conv_step", x.data_ptr(), x.stride(0), weight.data_ptr(), bias.data_ptr(), tail.data_ptr() or None,
          slots.data_ptr(), positions.data_ptr(), active.data_ptr(), out.data_ptr(), batch, tail.shape[0], channels, taps,
          _dtype(x))
    return out


def scan_dt(low: torch.Tensor, up: torch.Tensor, bias: torch.Tensor) -> torch.Tensor:
    """fp32 [rows, channels] = softplus(low up^T + bias); low [rows, rank] may be a view."""
    dev = _dev(up, bias)
    channels, rank = up.shape
    _rows_of(low, dev, rank)
    assert bias.shape == (channels,) and up.dtype == bias.dtype == low.dtype
    dt = torch.empty(low.shape[0], channels, dtype=torch.float32, device=dev)
    _call(dev, "nqh_scan_dt", low.data_ptr(), low.stride(0), up.data_ptr(), bias.data_ptr(), dt.data_ptr(), low.shape[0],
          channels, rank, _dtype(low))
    return dt


def _scan_args(x, dt, bc, z, a_log, skip, state):
    dev = _dev(x, dt, a_log, skip, state)
    channels, states = a_log.shape
    rows = x.shape[0]
    _rows_of(bc, dev, 2 * states)
    _rows_of(z, dev, channels)
    assert x.shape == (rows, channels) and dt.shape == (rows, channels) and dt.dtype == torch.float32
    assert bc.shape[0] == rows and z.shape[0] == rows and skip.shape == (channels,)
    assert x.dtype == bc.dtype == z.dtype == a_log.dtype == skip.dtype
    assert state.dtype == torch.float32 and state.shape[1:] == (states, channels)
    return dev, rows, channels, states, (x.data_ptr(), dt.data_ptr(), bc.data_ptr(), bc.stride(0), z.data_ptr(), z.stride(0),
                                         a_log.data_ptr(), skip.data_ptr())


def scan_prefill(x: torch.Tensor, dt: torch.Tensor, bc: torch.Tensor, z: torch.Tensor, a_log: torch.Tensor,
                 skip: torch.Tensor, conv_in: torch.Tensor, state: torch.Tensor, tail: torch.Tensor, layout: PromptPass,
                 piece_rows: int) -> torch.Tensor:
    """The pass's tokens through the recurrence: x, dt [rows, channels], bc [rows, B | C], z [rows, channels] (views).  state
    [slots, states, channels] and tail [slots, taps - 1, channels] (the convolution's last inputs, from conv_in) are moved on
    IN PLACE at the segments' slots.  Returns (y + skip x) silu(z) [rows, channels]."""
    dev, rows, channels, states, args = _scan_args(x, dt, bc, z, a_log, skip, state)
    _dev(state, tail)
    _rows_of(conv_in, dev, channels)
    assert rows == layout.rows and conv_in.shape[0] == rows and conv_in.dtype == x.dtype
    assert tail.dtype == torch.float32 and tail.shape[0] == state.shape[0] and tail.shape[2] == channels
    assert all(0 <= s[3] < state.shape[0] for s in layout.segments)
    assert piece_rows >= scan_piece_rows(1, channels, states)
    pieces, n, chained = layout.pieces(piece_rows)
    nbytes = _lib.hybrid_lib().nqh_scan_workspace_bytes(n, channels, states) if chained else 0
    ws = torch.empty(nbytes, dtype=torch.uint8, device=dev) if nbytes else None
    out = torch.empty(rows, channels, dtype=x.dtype, device=dev)
    _call(dev, "nqh_scan_prefill", *args, conv_in.data_ptr(), conv_in.stride(0), state.data_ptr(), tail.data_ptr() or None,
          pieces.data_ptr(), n, int(chained), out.data_ptr(), channels, states, tail.shape[1] + 1, _dtype(x), _ptr(ws), nbytes)
    return out


def scan_step(x: torch.Tensor, dt: torch.Tensor, bc: torch.Tensor, z: torch.Tensor, a_log: torch.Tensor, skip: torch.Tensor,
              state: torch.Tensor, slots: torch.Tensor, positions: torch.Tensor, active: torch.Tensor) -> torch.Tensor:
    """The same for one token per sequence, state IN PLACE at the rows' slots.  Idle rows change no state and give zeros."""
    dev, batch, channels, states, args = _scan_args(x, dt, bc, z, a_log, skip, state)
    _dev(state, slots, positions, active)
    assert slots.dtype == torch.int32 and positions.dtype == torch.int64 and active.dtype == torch.bool
    assert slots.numel() == batch and positions.numel() == batch and active.numel() == batch
    out = torch.empty(batch, channels, dtype=x.dtype, device=dev)
    _call(dev, "nqh_scan_step", *args, state.data_ptr(), slots.data_ptr(), positions.data_ptr(), active.data_ptr(),
          out.data_ptr(), batch, state.shape[0], channels, states, _dtype(x))
    return out


def _gla_offsets(proj: torch.Tensor, heads: int, dim: int, vdim: int, rank: int):
    """Addresses of q | k | v | gate | low in the rows of a projection."""
    nk, nv = heads * dim, heads * vdim
    assert proj.shape[1] == 2 * nk + 2 * nv + rank
    size, base = proj.element_size(), proj.data_ptr()
    return [base + size * o for o in (0, nk, 2 * nk, 2 * nk + nv, 2 * nk + 2 * nv)]


def gla_decay(proj: torch.Tensor, up: torch.Tensor, bias: torch.Tensor, heads: int, dim: int, vdim: int,
              tau: float) -> torch.Tensor:
    """fp32 [rows, heads * dim] = sigmoid(low up^T + bias)^(1 / tau), low being the last columns of the projection rows."""
    dev = _dev(proj, up, bias)
    channels, rank = up.shape
    assert channels == heads * dim and bias.shape == (channels,) and up.dtype == proj.dtype and bias.dtype == proj.dtype
    low = _gla_offsets(proj, heads, dim, vdim, rank)[4]
    decay = torch.empty(proj.shape[0], channels, dtype=torch.float32, device=dev)
    _call(dev, "nqh_gla_decay", low, proj.shape[1], up.data_ptr(), bias.data_ptr(), decay.data_ptr(), proj.shape[0],
          channels, rank, tau, _dtype(proj))
    return decay


def gla_prefill(proj: torch.Tensor, decay: torch.Tensor, state: torch.Tensor, layout: PromptPass, heads: int, dim: int,
                vdim: int, rank: int) -> torch.Tensor:
    """The tokens of the pass through the recurrence: state fp32 [slots, heads, dim, vdim] IN PLACE at the segments' slots
    (zero before position 0 whatever a slot holds); returns the read-outs, fp32 [rows, heads * vdim]."""
    dev = _dev(proj, decay, state, layout.tables)
    rows = proj.shape[0]
    assert rows == layout.rows and state.dtype == torch.float32 and state.shape[1:] == (heads, dim, vdim)
    assert all(0 <= s[3] < state.shape[0] for s in layout.segments)
    assert decay.shape == (rows, heads * dim) and decay.dtype == torch.float32
    q, k, v, _, _ = _gla_offsets(proj, heads, dim, vdim, rank)
    pieces, n, chained = layout.pieces(_lib.hybrid_lib().nqh_gla_piece_rows(rows, heads, dim, vdim))
    nbytes = _lib.hybrid_lib().nqh_gla_prefill_workspace_bytes(n, heads, dim, vdim) if chained else 0
    ws = torch.empty(nbytes, dtype=torch.uint8, device=dev) if nbytes else None
    o = torch.empty(rows, heads * vdim, dtype=torch.float32, device=dev)
    _call(dev, "nqh_gla_prefill", q, k, v, proj.shape[1], decay.data_ptr(), state.data_ptr(), o.data_ptr(), pieces.data_ptr(),
          n, int(chained), heads, dim, vdim, dim ** -0.5, _dtype(proj), _ptr(ws), nbytes)
    return o


def head_norm_gate(o: torch.Tensor, proj: torch.Tensor, weight: torch.Tensor, heads: int, dim: int, vdim: int, rank: int,
                   eps: float) -> torch.Tensor:
    """RMSNorm of o fp32 [rows, heads * vdim] per head, times weight [vdim], times SiLU(gate columns of proj)."""
    dev = _dev(o, proj, weight)
    rows = o.shape[0]
    assert o.dtype == torch.float32 and o.shape[1] == heads * vdim and proj.shape[0] == rows
    assert weight.shape == (vdim,) and weight.dtype == proj.dtype
    gate = _gla_offsets(proj, heads, dim, vdim, rank)[3]
    out = torch.empty(rows, heads * vdim, dtype=proj.dtype, device=dev)
    _call(dev, "nqh_head_norm_gate", o.data_ptr(), gate, proj.shape[1], weight.data_ptr(), out.data_ptr(), rows, heads, vdim,
          eps, _dtype(proj))
    return out


def gla_decode(proj: torch.Tensor, up: torch.Tensor, bias: torch.Tensor, norm_weight: torch.Tensor, state: torch.Tensor,
               slots: torch.Tensor, positions: torch.Tensor, active: torch.Tensor, heads: int, dim: int, vdim: int,
               tau: float, eps: float) -> torch.Tensor:
    """One token of each sequence: proj [batch, ...] rows, state [slots, heads, dim, vdim] fp32 IN PLACE at the rows'
    slots int32 [batch].  Idle rows (active false) change no state and give zeros.  Returns [batch, heads * vdim]."""
    dev = _dev(proj, up, bias, norm_weight, state, slots, positions, active)
    batch, rank = proj.shape[0], up.shape[1]
    assert up.shape[0] == heads * dim and bias.shape == (heads * dim,) and norm_weight.shape == (vdim,)
    assert up.dtype == proj.dtype and bias.dtype == proj.dtype and norm_weight.dtype == proj.dtype
    assert state.dtype == torch.float32 and state.shape[1:] == (heads, dim, vdim)
    assert slots.dtype == torch.int32 and positions.dtype == torch.int64 and active.dtype == torch.bool
    assert slots.numel() == batch and positions.numel() == batch and active.numel() == batch
    q, k, v, gate, low = _gla_offsets(proj, heads, dim, vdim, rank)
    out = torch.empty(batch, heads * vdim, dtype=proj.dtype, device=dev)
    _call(dev, "nqh_gla_decode", q, k, v, gate, low, proj.shape[1], up.data_ptr(), bias.data_ptr(), norm_weight.data_ptr(),
          state.data_ptr(), slots.data_ptr(), positions.data_ptr(), active.data_ptr(), out.data_ptr(), batch,
          state.shape[0], heads, dim, vdim, rank, tau, dim ** -0.5, eps, _dtype(proj))
    return out


def router_topk(h: torch.Tensor, router: torch.Tensor, top: int) -> Tuple[torch.Tensor, torch.Tensor]:
    """(expert int32 [rows, top], score fp32 [rows, top]) of the `top` largest sigmoid scores, largest first."""
    dev = _dev(h, router)
    rows, width = h.shape
    experts = router.shape[0]
    assert router.shape == (experts, width) and router.dtype == h.dtype
    expert = torch.empty(rows, top, dtype=torch.int32, device=dev)
    weight = torch.empty(rows, top, dtype=torch.float32, device=dev)
    _call(dev, "nqh_router_topk", h.data_ptr(), router.data_ptr(), expert.data_ptr(), weight.data_ptr(), rows, width,
          experts, top, _dtype(h))
    return expert, weight


def moe_plan(expert: torch.Tensor, experts: int, tile_rows: int) -> Tuple[torch.Tensor, torch.Tensor]:
    """Pairs (row, choice) of expert int32 [rows, top] grouped by expert: (order int32 [pairs], tile list)."""
    dev = _dev(expert)
    assert expert.dtype == torch.int32
    pairs = expert.numel()
    max_tiles = _lib.hybrid_lib().nqh_moe_max_tiles(pairs, experts, tile_rows)
    order = torch.empty(pairs, dtype=torch.int32, device=dev)
    tiles = torch.empty(3 * max_tiles + 1, dtype=torch.int32, device=dev)
    _call(dev, "nqh_moe_plan", expert.data_ptr(), order.data_ptr(), tiles.data_ptr(), pairs, experts, tile_rows, max_tiles)
    return order, tiles


def route(h: torch.Tensor, router: torch.Tensor, top: int, ff: int) -> Routing:
    """Router and plan of the experts for normalised rows h."""
    rows, width = h.shape
    r = Routing(rows, router.shape[0], top, width, ff, _dtype(h), h.device)
    r.expert, r.weight = router_topk(h, router, top)
    r.order, r.tiles = moe_plan(r.expert, r.experts, r.tile_rows)
    return r


def moe_experts(h: torch.Tensor, gate_up: torch.Tensor, down: torch.Tensor, r: Routing) -> torch.Tensor:
    """y [rows, top, width]: the chosen experts' outputs for the input scaled by their weights, not yet summed."""
    dev = _dev(h, gate_up, down, r.expert, r.weight, r.order, r.tiles)
    rows, width = h.shape
    experts, ff = gate_up.shape[0], down.shape[2]
    assert gate_up.shape == (experts, 2 * ff, width) and down.shape == (experts, width, ff) and experts == r.experts
    assert gate_up.dtype == h.dtype and down.dtype == h.dtype and rows * r.top == r.pairs
    act = torch.empty(r.pairs, ff, dtype=h.dtype, device=dev)
    _call(dev, "nqh_moe_gate_up", h.data_ptr(), gate_up.data_ptr(), r.weight.data_ptr(), r.order.data_ptr(),
          r.tiles.data_ptr(), act.data_ptr(), r.pairs, r.top, experts, width, ff, r.tile_rows, r.max_tiles, _dtype(h))
    y = torch.empty(rows, r.top, width, dtype=h.dtype, device=dev)
    _call(dev, "nqh_moe_down", act.data_ptr(), down.data_ptr(), r.order.data_ptr(), r.tiles.data_ptr(), y.data_ptr(),
          r.pairs, experts, width, ff, r.tile_rows, r.max_tiles, _dtype(h))
    return y


def skinny_linear_supported(rows: int, weight: torch.Tensor) -> bool:
    return 1 <= rows <= SKINNY_ROWS and weight.dtype == torch.bfloat16 and weight.shape[1] % 8 == 0


def skinny_linear(x: torch.Tensor, weight: torch.Tensor, bias: Optional[torch.Tensor] = None,
                  out_f32: bool = False, activation: Optional[str] = None, param: float = 0.0) -> torch.Tensor:
    """activation(x [rows <= 64, in] bf16 @ weight [out, in]^T (+ bias)), bf16 or (out_f32) fp32 result."""
    dev = _dev(x, weight, bias)
    rows, n = x.shape
    assert weight.shape[1] == n and x.dtype == torch.bfloat16 and weight.dtype == torch.bfloat16
    assert bias is None or (bias.shape == (weight.shape[0],) and bias.dtype == torch.bfloat16)
    y = torch.empty(rows, weight.shape[0], dtype=torch.float32 if out_f32 else torch.bfloat16, device=dev)
    _call(dev, "nqh_skinny_linear", x.data_ptr(), weight.data_ptr(), _ptr(bias), y.data_ptr(), rows, weight.shape[0], n,
          int(out_f32), ACTIVATIONS[activation], param)
    return y


def argmax_rows(logits: torch.Tensor) -> torch.Tensor:
    """Greedy sampler: int64 [rows] index of the largest fp32 logit per row (lowest index among equal maxima)."""
    dev = _dev(logits)
    rows, vocab = logits.shape
    assert logits.dtype == torch.float32
    out = torch.empty(rows, dtype=torch.int64, device=dev)
    _call(dev, "nqh_argmax_rows", logits.data_ptr(), out.data_ptr(), rows, vocab)
    return out


def decode_prepare(positions: torch.Tensor, active: torch.Tensor, block_table: torch.Tensor, block_size: int):
    """positions int64 [rows], active bool [rows], block_table int32 [rows, max_blocks] -> (slots int64 [rows] with -1
    for idle rows, context_lens int32 [rows] = positions + 1)."""
    dev = _dev(positions, active, block_table)
    rows = positions.numel()
    assert positions.dtype == torch.int64 and active.dtype == torch.bool and block_table.dtype == torch.int32
    assert active.numel() == rows and block_table.dim() == 2 and block_table.shape[0] == rows
    slots = torch.empty(rows, dtype=torch.int64, device=dev)
    ctx = torch.empty(rows, dtype=torch.int32, device=dev)
    _call(dev, "nqh_decode_prepare", positions.data_ptr(), active.data_ptr(), block_table.data_ptr(), slots.data_ptr(),
          ctx.data_ptr(), rows, block_table.shape[1], block_size)
    return slots, ctx


def decode_advance(next_tokens: torch.Tensor, active: torch.Tensor, out_log: torch.Tensor, ids: torch.Tensor,
                   positions: torch.Tensor, step: torch.Tensor) -> None:
    """IN PLACE: out_log[step[0]] = next_tokens, ids = next_tokens, positions += active, step += 1."""
    dev = _dev(next_tokens, active, out_log, ids, positions, step)
    rows = next_tokens.numel()
    assert all(t.dtype == torch.int64 for t in (next_tokens, out_log, ids, positions, step)) and active.dtype == torch.bool
    assert out_log.dim() == 2 and out_log.shape[1] == rows and ids.numel() == rows and positions.numel() == rows
    assert active.numel() == rows and step.numel() == 1
    _call(dev, "nqh_decode_advance", next_tokens.data_ptr(), active.data_ptr(), out_log.data_ptr(), ids.data_ptr(),
          positions.data_ptr(), step.data_ptr(), rows, out_log.shape[0])
