"""Decoders described layer by layer: specifications and weights.

A DecoderSpec lists layers; each has a mixer (attention over the paged KV cache, attention over cached latents, gated linear
attention or a selective scan with a recurrent state), an optional feed-forward (dense or a mixture of experts), norms before
and possibly after both, and a residual that is one row per token or several streams.  Every constant is a field here, so a
design is a function from its configuration to a spec plus a table of checkpoint names (models/gafulix.py,
models/roletar.py); the engine (engine/hybrid_engine.py) reads the spec only.

Weights are held in the layout the kernels want: projections with a common input side by side in one matrix, the
experts of a layer stacked.  Checkpoint tensors are copied into views of those (`HybridDecoder.checkpoint_views`)."""
from __future__ import annotations

import math
from dataclasses import dataclass
from typing import Dict, List, Optional, Tuple, Union

import torch
from torch import nn


@dataclass(frozen=True)
class YarnScaling:
    """Frequencies divided by `factor` for the slow pairs, kept for the fast ones, ramped in between; `fast` and `slow`
    are numbers of rotations over `original` positions."""
    factor: float
    original: float
    fast: float
    slow: float


@dataclass(frozen=True)
class RotarySpec:
    """Rotary angles of the first `dims` dimensions of a head, pairs (2i, 2i + 1)."""
    dims: int
    base: float
    scaling: Optional[YarnScaling] = None


@dataclass(frozen=True)
class AttentionSpec:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rotary: Optional[RotarySpec] = None
    chunk: int = 0              # > 0: tokens see keys of their own chunk of that many positions only
    window: int = 0             # > 0: tokens see themselves and the window - 1 tokens before them
    sink: bool = False          # a learned score per head that takes part in the softmax without key or value
    bias: bool = True           # of the q, k and v projections
    qk_norm: bool = True        # RMS norm over the whole q and the whole k projection

    def __post_init__(self):
        if self.heads % self.kv_heads:
            raise ValueError(f"{self.heads} query heads do not divide over {self.kv_heads} key/value heads")


@dataclass(frozen=True)
class LatentAttentionSpec:
    """Keys and values of all heads come from one normalised latent of `rank` elements per token; a rotated key part of
    rotary.dims elements is shared by all heads.  Query heads are [dim | rotary.dims].  Latent and rotated part are what is
    cached."""
    heads: int
    dim: int
    vdim: int
    rank: int
    scale: float
    rotary: RotarySpec


@dataclass(frozen=True)
class SelectiveScanSpec:
    """S = exp(dt A) S + dt x B, y = S C + D x per channel, behind a causal convolution of `taps` tokens."""
    channels: int
    state: int
    dt_rank: int
    taps: int


@dataclass(frozen=True)
class GatedLinearSpec:
    """S = diag(decay) S + k v^T, o = S^T q, decay = sigmoid(low-rank projection)^(1 / tau) per key channel."""
    heads: int
    dim: int
    vdim: int
    tau: float
    rank: int


@dataclass(frozen=True)
class MoESpec:
    """Sigmoid router, `top` experts per token, the score multiplies the expert's input."""
    experts: int
    top: int
    ff: int


@dataclass(frozen=True)
class DenseSpec:
    """down act(up h); `activation` names one of engine/hybrid_ops.py ACTIVATIONS."""
    ff: int
    activation: str


@dataclass(frozen=True)
class LayerSpec:
    mixer: Union[AttentionSpec, LatentAttentionSpec, GatedLinearSpec, SelectiveScanSpec]
    mlp: Optional[Union[MoESpec, DenseSpec]]


@dataclass(frozen=True)
class LoopSpec:
    """Layers start .. stop - 1 run `times` times in a row; passes after the first add the embedding output first if
    `reinject`."""
    start: int
    stop: int
    times: int
    reinject: bool = True


@dataclass(frozen=True)
class DecoderSpec:
    vocab: int
    width: int
    eps: float
    layers: Tuple[LayerSpec, ...]
    loop: Optional[LoopSpec] = None
    post_norms: bool = True           # sublayer outputs are normalised before they are added
    streams: int = 0                  # > 0: hyper-connections over that many residual streams
    logit_cap: float = 0.0            # > 0: logits = cap * tanh(logits / cap)

    def __post_init__(self):
        lp = self.loop
        if lp is not None and not (0 <= lp.start < lp.stop <= len(self.layers) and lp.times >= 1):
            raise ValueError(f"loop {lp} does not fit {len(self.layers)} layers")
        if self.streams and (self.post_norms or any(again for _, again in self.runs())
                             or any(isinstance(l.mlp, MoESpec) for l in self.layers)):
            raise ValueError("residual streams go with pre-norm layers, dense feed-forwards and loops that add nothing")

    def runs(self) -> List[Tuple[int, bool]]:
        """(layer index, whether the embedding output is added in front of it) in execution order.  Every run has its
        own cache or state."""
        n, lp = len(self.layers), self.loop
        if lp is None:
            return [(i, False) for i in range(n)]
        out = [(i, False) for i in range(lp.start)]
        for rep in range(lp.times):
            out += [(i, lp.reinject and rep > 0 and i == lp.start) for i in range(lp.start, lp.stop)]
        return out + [(i, False) for i in range(lp.stop, n)]


def rotary_table(spec: RotarySpec, positions: int) -> torch.Tensor:
    """fp32 [positions, dims] = cos | sin of every pair's angle, the magnitude factor of a scaling included.  Computed in
    float64 and rounded once: at large positions a float32 product would already be off by several ulps of 2 pi."""
    d, base, sc = spec.dims, float(spec.base), spec.scaling
    i = torch.arange(d // 2, dtype=torch.float64)
    freq = base ** (-2.0 * i / d)
    magnitude = 1.0
    if sc is not None:
        def pair(turns: float) -> float:
            return d * math.log(sc.original / (2.0 * math.pi * turns)) / (2.0 * math.log(base))
        lo, hi = max(math.floor(pair(sc.fast)), 0), min(math.ceil(pair(sc.slow)), d - 1)
        ramp = ((i - lo) / max(hi - lo, 0.001)).clamp(0.0, 1.0)
        freq = freq / sc.factor * ramp + freq * (1.0 - ramp)
        magnitude = 0.1 * math.log(sc.factor) + 1.0
    angle = torch.arange(positions, dtype=torch.float64).unsqueeze(1) * freq
    return torch.cat([angle.cos() * magnitude, angle.sin() * magnitude], dim=1).float()


def _param(*shape: int) -> nn.Parameter:
    return nn.Parameter(torch.zeros(*shape), requires_grad=False)


class AttentionWeights(nn.Module):
    def __init__(self, spec: AttentionSpec, width: int):
        super().__init__()
        nq, nk, nv = spec.heads * spec.dim, spec.kv_heads * spec.dim, spec.kv_heads * spec.vdim
        self.splits = (nq, nk, nv)
        self.qkv = _param(nq + nk + nv, width)
        self.qkv_bias = _param(nq + nk + nv) if spec.bias else None
        self.q_norm, self.k_norm = (_param(nq), _param(nk)) if spec.qk_norm else (None, None)
        self.sink = _param(spec.heads) if spec.sink else None
        self.out = _param(width, spec.heads * spec.vdim)


class LatentAttentionWeights(nn.Module):
    def __init__(self, spec: LatentAttentionSpec, width: int):
        super().__init__()
        rot = spec.rotary.dims
        self.splits = (spec.heads * (spec.dim + rot), spec.rank + rot)       # queries | latent and rotated key part
        self.proj = _param(sum(self.splits), width)
        self.latent_norm = _param(spec.rank)
        self.expand = _param(spec.heads * (spec.dim + spec.vdim), spec.rank)      # unrotated keys of all heads | values
        self.out = _param(width, spec.heads * spec.vdim)
        self.key_rows, self.head_dims = spec.heads * spec.dim, (spec.heads, spec.dim, spec.vdim, spec.rank)

    def per_head(self) -> Tuple[torch.Tensor, torch.Tensor]:
        """(the key expansion transposed per head [heads, rank, dim], which takes a query into the latent space; the value
        expansion [heads, vdim, rank])."""
        H, dim, vdim, rank = self.head_dims
        keys, values = self.expand.split([H * dim, H * vdim])
        return keys.view(H, dim, rank).transpose(1, 2).contiguous(), values.view(H, vdim, rank)


class SelectiveScanWeights(nn.Module):
    def __init__(self, spec: SelectiveScanSpec, width: int):
        super().__init__()
        C, N, rank = spec.channels, spec.state, spec.dt_rank
        self.proj = _param(2 * C, width)                                 # x | z
        self.conv, self.conv_bias = _param(C, spec.taps), _param(C)
        self.select = _param(rank + 2 * N, C)                            # dt | B | C
        self.dt_up, self.dt_bias = _param(C, rank), _param(C)
        self.a_log, self.skip = _param(C, N), _param(C)
        self.out = _param(width, C)


class GatedLinearWeights(nn.Module):
    def __init__(self, spec: GatedLinearSpec, width: int):
        super().__init__()
        nk, nv = spec.heads * spec.dim, spec.heads * spec.vdim
        self.splits = (nk, nk, nv, nv, spec.rank)          # q | k | v | gate | low-rank decay input
        self.proj = _param(sum(self.splits), width)
        self.decay_up, self.decay_bias = _param(nk, spec.rank), _param(nk)
        self.head_norm = _param(spec.vdim)
        self.out = _param(width, nv)


class MoEWeights(nn.Module):
    def __init__(self, spec: MoESpec, width: int):
        super().__init__()
        self.router = _param(spec.experts, width)
        self.gate_up = _param(spec.experts, 2 * spec.ff, width)
        self.down = _param(spec.experts, width, spec.ff)


class DenseWeights(nn.Module):
    def __init__(self, spec: DenseSpec, width: int):
        super().__init__()
        self.up, self.down = _param(spec.ff, width), _param(width, spec.ff)


class StreamWeights(nn.Module):
    """Hyper-connection of a sublayer: what it reads of every stream, how the old streams [from, to] and its output make the
    new ones."""

    def __init__(self, streams: int):
        super().__init__()
        self.read, self.write, self.mix = _param(streams), _param(streams), _param(streams, streams)


WEIGHTS = {AttentionSpec: AttentionWeights, LatentAttentionSpec: LatentAttentionWeights, GatedLinearSpec: GatedLinearWeights,
           SelectiveScanSpec: SelectiveScanWeights, MoESpec: MoEWeights, DenseSpec: DenseWeights}


class HybridLayer(nn.Module):
    def __init__(self, spec: LayerSpec, width: int, post_norms: bool, streams: int):
        super().__init__()
        def norms():
            return _param(width), _param(width) if post_norms else None
        self.norm_mixer, self.norm_mixer_out = norms()
        self.mixer = WEIGHTS[type(spec.mixer)](spec.mixer, width)
        self.mixer_streams = StreamWeights(streams) if streams else None
        self.mlp = self.mlp_streams = None
        if spec.mlp is not None:
            self.norm_mlp, self.norm_mlp_out = norms()
            self.mlp = WEIGHTS[type(spec.mlp)](spec.mlp, width)
            self.mlp_streams = StreamWeights(streams) if streams else None

    def linears(self) -> List[torch.Tensor]:
        """The matrices of this layer's plain products."""
        out = [w for n in ("qkv", "proj", "select", "out") if (w := getattr(self.mixer, n, None)) is not None]
        return out + ([self.mlp.up, self.mlp.down] if isinstance(self.mlp, DenseWeights) else [])


class HybridDecoder(nn.Module):
    """Weights of a DecoderSpec.  The forward pass is the engine's."""

    def __init__(self, spec: DecoderSpec):
        super().__init__()
        self.spec = spec
        self.embed = _param(spec.vocab, spec.width)
        self.layers = nn.ModuleList([HybridLayer(l, spec.width, spec.post_norms, spec.streams) for l in spec.layers])
        self.final_norm = _param(spec.width)
        self.head = _param(spec.vocab, spec.width)

    def checkpoint_views(self) -> Dict[str, torch.Tensor]:
        """Checkpoint tensor name -> the (view of a) parameter it fills.  Supplied by the design."""
        raise NotImplementedError

    def ignores(self, name: str) -> bool:
        """Whether a checkpoint may hold `name` although the model has no use for it."""
        return False
