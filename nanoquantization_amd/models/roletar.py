"""Roletar: a decoder of sliding-window attention with sinks, latent attention and selective-scan layers with squared-relu
feed-forwards, a residual of several streams joined by hyper-connections, capped logits and an optional loop over a range of
layers.  Configuration and checkpoint names; the mechanisms are those of models/hybrid.py and engine/hybrid_engine.py."""
from __future__ import annotations

from typing import Dict, Optional, Tuple

import torch

from .hybrid import (AttentionSpec, DecoderSpec, DenseSpec, HybridDecoder, LatentAttentionSpec, LayerSpec, LoopSpec, RotarySpec,
                     SelectiveScanSpec)

ARCHITECTURE = "Roletar"


def _mixer(kind: str, cfg: dict):
    if kind == "attention":
        return AttentionSpec(heads=cfg["heads"], kv_heads=cfg["kv_heads"], dim=cfg["dim"], vdim=cfg["vdim"],
                             scale=float(cfg["scale"]), window=int((cfg.get("mask") or {}).get("size") or 0), sink=True,
                             bias=False, qk_norm=False)
    if kind == "latent_attention":
        rot = cfg["rot"]
        if rot["dims"] != cfg["rot_dim"]:
            raise ValueError(f"{rot['dims']} rotated dimensions, but {cfg['rot_dim']} in the rotated part of a head")
        return LatentAttentionSpec(heads=cfg["heads"], dim=cfg["dim"], vdim=cfg["vdim"], rank=cfg["kv_rank"],
                                   scale=float(cfg["scale"]), rotary=RotarySpec(int(rot["dims"]), float(rot["base"])))
    if kind == "mamba1":
        return SelectiveScanSpec(channels=cfg["inner"], state=cfg["state"], dt_rank=cfg["dt_rank"], taps=cfg["conv"])
    raise ValueError(f"unknown mixer type {kind!r}")


def _mlp(cfg: Optional[dict]) -> Optional[DenseSpec]:
    if not cfg:
        return None
    if cfg.get("kind", "dense") != "dense":
        raise ValueError(f"unknown feed-forward kind {cfg['kind']!r}")
    return DenseSpec(ff=cfg["ff"], activation="relu2")


def spec_from_config(cfg: dict, shapes: Optional[Dict[str, Tuple[int, ...]]] = None) -> DecoderSpec:
    lp = cfg.get("loop")
    return DecoderSpec(vocab=cfg["vocab"], width=cfg["width"], eps=float(cfg["norm"]["eps"]),
                       layers=tuple(LayerSpec(_mixer(l["type"], l["mixer"]), _mlp(l.get("mlp"))) for l in cfg["layers"]),
                       loop=None if not lp else LoopSpec(lp["start"], lp["stop"], lp["times"], reinject=False),
                       post_norms=False, streams=int(cfg["streams"]), logit_cap=float(cfg.get("logit_softcap") or 0.0))


class RoletarForCausalLM(HybridDecoder):
    def checkpoint_views(self) -> Dict[str, torch.Tensor]:
        views = {"embed": self.embed, "final.norm": self.final_norm, "head": self.head}
        for i, (layer, spec) in enumerate(zip(self.layers, self.spec.layers)):
            p, mix, m = f"l{i}.", layer.mixer, spec.mixer
            views[p + "norm1"] = layer.norm_mixer
            named = {"o": mix.out}
            if isinstance(m, AttentionSpec):
                named.update(zip("qkv", mix.qkv.split(mix.splits)), sink=mix.sink)
            elif isinstance(m, LatentAttentionSpec):
                named.update(zip(("q", "dkv"), mix.proj.split(mix.splits)))
                named.update({"dkv.norm": mix.latent_norm, "uk": mix.expand[:mix.key_rows], "uv": mix.expand[mix.key_rows:]})
            else:
                named.update({"in": mix.proj, "conv": mix.conv, "conv.b": mix.conv_bias, "x": mix.select, "dt": mix.dt_up,
                              "dt.b": mix.dt_bias, "A_log": mix.a_log, "D": mix.skip})
            views.update({f"{p}mix.{n}": t for n, t in named.items()})
            if layer.mlp is not None:
                views[p + "norm2"] = layer.norm_mlp
                views[p + "mlp.up"], views[p + "mlp.down"] = layer.mlp.up, layer.mlp.down
            for n, hc in (("1", layer.mixer_streams), ("2", layer.mlp_streams)):
                if hc is not None:
                    views[f"{p}hc{n}.in"], views[f"{p}hc{n}.out"], views[f"{p}hc{n}.mix"] = hc.read, hc.write, hc.mix
        return views

    def ignores(self, name: str) -> bool:
        # what would belong to the feed-forward of a layer that has none
        head, _, tail = name.partition(".")
        return ((tail == "norm2" or tail.startswith("hc2.")) and head[:1] == "l" and head[1:].isdigit()
                and int(head[1:]) < len(self.layers) and self.layers[int(head[1:])].mlp is None)
