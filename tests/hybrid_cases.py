"""Small random configurations and weights of hybrid decoders, shared by the tests."""
import torch

ATT = dict(type="attention", mixer=dict(heads=6, kv_heads=2, dim=40, vdim=24, scale=0.21, mask=dict(size=20),
                                        rot=dict(base=500.0, dims=24, scaling=dict(factor=3.0, original=64, fast=8.0,
                                                                                   slow=0.5))),
           mlp=dict(kind="moe", expert=dict(ff=48), router=dict(experts=5, top=2)))
GLA = dict(type="gla", mixer=dict(heads=3, dim=24, vdim=40, tau=4.0),
           mlp=dict(kind="moe", expert=dict(ff=24), router=dict(experts=7, top=3)))


def layer(base, mlp="keep", **mixer):
    out = dict(type=base["type"], mixer=dict(base["mixer"], **mixer), mlp=base["mlp"] if mlp == "keep" else mlp)
    return out


def config(layers, loop=None, vocab=131, width=72, eps=1e-5):
    return dict(architecture="Gafulix", layers=layers, loop=loop, norm=dict(eps=eps), vocab=vocab, width=width)


# name -> configuration; sizes that are not powers of two, dim != vdim, partial rotation, every branch on and off; widths
# that are and are not multiples of 8 (matrix-core kernels or not), many query heads on one key/value head
CONFIGS = {
    "loop_middle": config([layer(GLA), layer(ATT), layer(GLA, tau=1.0, heads=2, dim=16, vdim=16),
                           layer(ATT, mask=dict(size=33), heads=4, kv_heads=4)], dict(start=1, stop=3, times=3)),
    "no_loop": config([layer(ATT, rot=dict(base=10000.0, dims=40, scaling=None), heads=4, kv_heads=1),
                       layer(GLA, mlp=None, dim=22, vdim=26), layer(ATT, mlp=None, mask=dict(size=7))], vocab=97, width=68),
    "loop_all": config([layer(ATT, dim=64, vdim=96, heads=2, kv_heads=1, mask=dict(size=48),
                              mlp=dict(kind="moe", expert=dict(ff=64), router=dict(experts=9, top=1))),
                        layer(GLA, heads=2, dim=64, vdim=48, tau=16.0)], dict(start=0, stop=2, times=2), width=128),
    "many_heads": config([layer(ATT, heads=20, kv_heads=1, dim=16, vdim=32, rot=None, mask=dict(size=30)),
                          layer(GLA, heads=5, dim=48, vdim=16, tau=2.0,
                                mlp=dict(kind="moe", expert=dict(ff=16), router=dict(experts=150, top=5)))],
                         vocab=200, width=80),
    "one_pass_loop": config([layer(GLA, mlp=dict(kind="moe", expert=dict(ff=32), router=dict(experts=4, top=4))),
                             layer(ATT, mask=dict(size=64), dim=32, vdim=32, heads=8, kv_heads=2)],
                            dict(start=1, stop=2, times=1), width=96, eps=1e-3),
}


# Roletar: sliding windows with sinks, latent attention, selective scans, several residual streams
WIN = dict(type="attention", mixer=dict(heads=6, kv_heads=3, dim=40, vdim=24, scale=0.23, mask=dict(size=17)),
           mlp=dict(kind="dense", ff=88))
LATENT = dict(type="latent_attention", mixer=dict(heads=5, dim=24, rot_dim=8, vdim=40, kv_rank=72, scale=0.19,
                                                  rot=dict(base=700.0, dims=8)), mlp=dict(kind="dense", ff=64))
SCAN = dict(type="mamba1", mixer=dict(inner=88, state=24, dt_rank=8, conv=4), mlp=None)


def latent(mlp="keep", rot_dim=8, base=700.0, **mixer):
    return layer(LATENT, mlp, rot_dim=rot_dim, rot=dict(base=base, dims=rot_dim), **mixer)


def roletar(layers, loop=None, vocab=131, width=72, eps=1e-5, streams=2, cap=12.0):
    return dict(architecture="Roletar", layers=layers, loop=loop, norm=dict(eps=eps), vocab=vocab, width=width,
                streams=streams, logit_softcap=cap)


# every kind of layer with and without a feed-forward, widths that are and are not multiples of 8, one to eight streams, a
# window of one, state sizes for one lane and for sixteen per channel, one to seven taps, latents for every kernel form
CONFIGS.update({
    "roletar_loop_middle": roletar([layer(SCAN, mlp=WIN["mlp"]), layer(WIN), latent(mlp=None), layer(SCAN, state=16),
                                    layer(WIN, mlp=None, mask=dict(size=33), heads=4, kv_heads=4), latent(kv_rank=40)],
                                   dict(start=1, stop=4, times=3), streams=3),
    "roletar_one_stream": roletar([layer(WIN, mask=dict(size=1), dim=22, vdim=18, heads=4, kv_heads=2),
                                   layer(SCAN, inner=50, state=5, dt_rank=3, conv=2),
                                   latent(kv_rank=50, rot_dim=6, dim=22, vdim=26, heads=3)], width=68, vocab=97, streams=1),
    "roletar_wide": roletar([latent(kv_rank=264, rot_dim=64, dim=128, vdim=96, heads=18, scale=0.07),
                             layer(SCAN, inner=64, state=130, dt_rank=16, conv=1, mlp=LATENT["mlp"]),
                             layer(WIN, dim=64, vdim=96, heads=4, kv_heads=1, mask=dict(size=48))],
                            dict(start=0, stop=3, times=2), width=128, streams=5, cap=3.0),
    "roletar_many": roletar([layer(SCAN, inner=320, state=33, dt_rank=24, conv=7),
                             layer(WIN, heads=20, kv_heads=1, dim=16, vdim=32, mask=None),
                             latent(kv_rank=128, rot_dim=32, dim=32, vdim=160, heads=2)],
                            dict(start=1, stop=2, times=1), vocab=200, width=80, streams=8, eps=1e-3, cap=40.0),
    "roletar_no_state": roletar([latent(rot_dim=40, kv_rank=200), layer(WIN, mlp=None)], width=64, streams=4),
})


def _gafulix_shapes(cfg, rank):
    D, shapes = cfg["width"], {"embed": (cfg["vocab"], cfg["width"]), "final.norm": (cfg["width"],),
                               "head": (cfg["vocab"], cfg["width"])}
    for i, l in enumerate(cfg["layers"]):
        m, p = l["mixer"], f"l{i}."
        for n in ("norm1", "norm1b") + (("norm2", "norm2b") if l["mlp"] else ()):
            shapes[p + n] = (D,)
        if l["type"] == "attention":
            nq, nk, nv = m["heads"] * m["dim"], m["kv_heads"] * m["dim"], m["kv_heads"] * m["vdim"]
            for n, s in (("q", nq), ("k", nk), ("v", nv)):
                shapes[f"{p}mix.{n}"], shapes[f"{p}mix.{n}.b"] = (s, D), (s,)
            shapes[p + "mix.q.norm"], shapes[p + "mix.k.norm"] = (nq,), (nk,)
            shapes[p + "mix.o"] = (D, m["heads"] * m["vdim"])
        else:
            nk, nv = m["heads"] * m["dim"], m["heads"] * m["vdim"]
            for n, s in (("q", nk), ("k", nk), ("v", nv), ("g", nv), ("a1", rank)):
                shapes[f"{p}mix.{n}"] = (s, D)
            shapes[p + "mix.a2"], shapes[p + "mix.a2.b"] = (nk, rank), (nk,)
            shapes[p + "mix.norm"], shapes[p + "mix.o"] = (m["vdim"],), (D, nv)
        if l["mlp"]:
            ff, experts = l["mlp"]["expert"]["ff"], l["mlp"]["router"]["experts"]
            shapes[p + "mlp.router"] = (experts, D)
            for e in range(experts):
                shapes[f"{p}mlp.e{e}.gate"] = shapes[f"{p}mlp.e{e}.up"] = (ff, D)
                shapes[f"{p}mlp.e{e}.down"] = (D, ff)
    return shapes


def _roletar_shapes(cfg):
    D, S, shapes = cfg["width"], cfg["streams"], {"embed": (cfg["vocab"], cfg["width"]), "final.norm": (cfg["width"],),
                                                  "head": (cfg["vocab"], cfg["width"])}
    for i, l in enumerate(cfg["layers"]):
        m, p = l["mixer"], f"l{i}."
        for n in ("1", "2") if l["mlp"] else ("1",):
            shapes.update({f"{p}norm{n}": (D,), f"{p}hc{n}.in": (S,), f"{p}hc{n}.out": (S,), f"{p}hc{n}.mix": (S, S)})
        if l["type"] == "attention":
            H, G = m["heads"], m["kv_heads"]
            mix = {"q": (H * m["dim"], D), "k": (G * m["dim"], D), "v": (G * m["vdim"], D), "sink": (H,), "o": (D, H * m["vdim"])}
        elif l["type"] == "latent_attention":
            H, rank, rot = m["heads"], m["kv_rank"], m["rot_dim"]
            mix = {"q": (H * (m["dim"] + rot), D), "dkv": (rank + rot, D), "dkv.norm": (rank,), "uk": (H * m["dim"], rank),
                   "uv": (H * m["vdim"], rank), "o": (D, H * m["vdim"])}
        else:
            C, N, rank = m["inner"], m["state"], m["dt_rank"]
            mix = {"in": (2 * C, D), "conv": (C, m["conv"]), "conv.b": (C,), "x": (rank + 2 * N, C), "dt": (C, rank),
                   "dt.b": (C,), "A_log": (C, N), "D": (C,), "o": (D, C)}
        shapes.update({p + "mix." + n: s for n, s in mix.items()})
        if l["mlp"]:
            shapes[p + "mlp.up"], shapes[p + "mlp.down"] = (l["mlp"]["ff"], D), (D, l["mlp"]["ff"])
    return shapes


def tensor_shapes(cfg, rank=16):
    return _roletar_shapes(cfg) if cfg["architecture"] == "Roletar" else _gafulix_shapes(cfg, rank)


_per_input = lambda gain: lambda t: t * gain * t.shape[-1] ** -0.5
# squared activations and repeated passes amplify rounding: gains low enough that bf16 is not chaotic
_ROLETAR_INIT = {"sink": lambda t: 2.0 + t, "A_log": lambda t: torch.arange(1.0, t.shape[1] + 1).log() - 2.0 + 0.5 * t,
                 "D": lambda t: 1.0 + 0.5 * t, "in": lambda t: _per_input(1.0)(t) if t.dim() == 2 else 0.5 + 0.2 * t,
                 "out": lambda t: 0.6 + 0.3 * t, "mix": lambda t: torch.eye(len(t)) + 0.1 * t, "up": _per_input(1.0),
                 "down": _per_input(0.4), "uk": _per_input(1.0), "o": _per_input(1.0)}


def random_weights(cfg, seed=0, rank=16, clear_routing=False):
    """bf16 weights: linears that keep their input's scale, norm weights around 1, biases and decays that matter.
    `clear_routing`: the first 8 dimensions hold the token's class, no sublayer writes them and the routers read nothing
    else, so that no choice of an expert is a close call that bf16 rounding could turn over."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(cfg, rank).items():
        t = torch.randn(shape, generator=g)
        last = name.split(".")[-1]
        if "norm" in last:
            t = 1.0 + 0.3 * t
        elif cfg["architecture"] == "Roletar" and last in _ROLETAR_INIT:
            t = _ROLETAR_INIT[last](t)
        elif name.endswith("dt.b"):
            t = t - 1.5                             # memories of a few tokens and of hundreds
        elif last == "b":
            t = t + 2.0 if ".a2." in name else 0.3 * t
        elif name == "embed":
            pass
        elif last == "router":
            t = t * 2.0 / shape[-1] ** 0.5          # far apart: a choice is never a close call
        else:
            t = t * 1.4 / shape[-1] ** 0.5
        if clear_routing:
            if name == "embed":
                t[:, :8] = 3.0 * torch.eye(8)[torch.arange(shape[0]) % 8]
            elif last in ("o", "down"):
                t[:8] = 0
            elif last == "router":
                t = torch.zeros(shape)
                for c in range(8):
                    t[:, c] = torch.linspace(-1.0, 0.5, shape[0])[torch.randperm(shape[0], generator=g)]
            elif last in ("norm1b", "norm2b", "norm2"):
                t = t.abs()
        out[name] = t.to(torch.bfloat16)
    return out


def write_checkpoint(path, cfg, weights):
    import json
    from safetensors.torch import save_file
    save_file(weights, str(path / "model.safetensors"))
    with open(path / "config.json", "w") as f:
        json.dump(cfg, f)


def tokens(n, vocab, seed=1):
    return torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def logit_error(got, want):
    """Worst row: rms over the vocabulary of the difference (mean taken off) against the rms spread of the expected
    logits."""
    got, want = got.double().cpu(), want.double().cpu()
    d = got - want
    d = d - d.mean(dim=-1, keepdim=True)
    scale = (want - want.mean(dim=-1, keepdim=True)).pow(2).mean().sqrt()
    return (d.pow(2).mean(dim=-1).sqrt() / scale).max().item()
