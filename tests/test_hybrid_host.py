"""Hybrid decoders without a GPU: configuration, checkpoint layout, rotary table, cache and state bookkeeping, the
library's exported symbols and argument checks, and the oracle's own consistency."""
import ctypes
import json
import os
import re

import pytest
import torch

from hybrid_cases import (ATT, CONFIGS, GLA, LATENT, WIN, config, latent, layer, random_weights, roletar, tensor_shapes, tokens,
                          write_checkpoint)
from nanoquantization_amd import _lib
from nanoquantization_amd.engine.cache import PagedKVCache, RecurrentStateCache
from nanoquantization_amd.models import registry
from nanoquantization_amd.models.gafulix import GafulixForCausalLM, spec_from_config
from nanoquantization_amd.models.hybrid import DecoderSpec, RotarySpec, YarnScaling, rotary_table
from nanoquantization_amd.models.roletar import spec_from_config as roletar_spec
from nanoquantization_amd.utils.loader import model_from_config, save_views
from oracle import hybrid_oracle as o

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


def test_library_exports_every_declared_symbol():
    if not os.path.exists(_lib.HYBRID_LIB_PATH):
        from nanoquantization_amd.build import build_hybrid
        build_hybrid(verbose=False)
    header = open(os.path.join(ROOT, "include", "nq_hybrid_ops.h")).read()
    declared = set(re.findall(r"\b(nqh_[a-z0-9_]+)\s*\(", header))
    handle = ctypes.CDLL(_lib.HYBRID_LIB_PATH)
    for name in sorted(declared):
        assert hasattr(handle, name), f"{name} declared but not exported"
    assert declared == set(_lib.HYBRID_SYMBOLS), "ctypes table and header disagree"
    L = _lib.hybrid_lib()
    assert L.nqh_argmax_rows(None, None, 1, 1, None) == 1 and b"null" in L.nqh_last_error()
    with pytest.raises(_lib.AwqHipError, match="nqh_moe_plan"):
        _lib.check_hybrid(L.nqh_moe_plan(None, None, None, 1, 1, 1, 1, None))
    for pairs, experts, rows in ((1, 1, 16), (5, 8, 16), (100, 3, 32), (64, 64, 16)):
        # the worst split: one pair in all experts but one
        worst = 0
        for used in range(1, min(pairs, experts) + 1):
            worst = max(worst, (used - 1) + -(-(pairs - used + 1) // rows))
        assert L.nqh_moe_max_tiles(pairs, experts, rows) >= worst


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_checkpoint_round_trip_and_views(name, tmp_path):
    cfg, w = CONFIGS[name], random_weights(CONFIGS[name], rank=12)
    write_checkpoint(tmp_path, cfg, w)
    m = model_from_config(str(tmp_path))
    assert type(m).__name__ == cfg["architecture"] + "ForCausalLM"
    views = m.checkpoint_views()
    assert {k: tuple(v.shape) for k, v in views.items()} == {k: tuple(s) for k, s in tensor_shapes(cfg, 12).items()}
    for k, v in views.items():
        assert torch.equal(v, w[k]), k
    out = tmp_path / "again"
    save_views(m, str(out), cfg)
    m2 = model_from_config(str(out), dtype=torch.float32)
    for k, v in m2.checkpoint_views().items():
        assert v.dtype == torch.float32 and torch.equal(v, w[k].float()), k


def test_loader_rejects_what_does_not_fit(tmp_path):
    cfg = CONFIGS["no_loop"]
    w = random_weights(cfg)
    for change, error in ((lambda d: d.pop("l1.mix.norm"), ValueError),
                          (lambda d: d.update({"l0.mix.extra": torch.zeros(1)}), AttributeError),
                          (lambda d: d.update({"l0.mix.o": torch.zeros(3, 3)}), ValueError)):
        bad = dict(w)
        change(bad)
        write_checkpoint(tmp_path, cfg, bad)
        with pytest.raises(error):
            model_from_config(str(tmp_path))
    ok = dict(w)
    ok["l1.norm2"] = ok["l1.norm2b"] = torch.ones(cfg["width"], dtype=torch.bfloat16)    # layer 1 has no feed-forward
    write_checkpoint(tmp_path, cfg, {k: v.clone() for k, v in ok.items()})
    model_from_config(str(tmp_path))


def test_roletar_configuration(tmp_path):
    cfg = CONFIGS["roletar_loop_middle"]
    spec = roletar_spec(cfg)
    assert spec.runs() == [(i, False) for i in (0, 1, 2, 3, 1, 2, 3, 1, 2, 3, 4, 5)] and o.layer_schedule(cfg)[4] == (1, True)
    assert (spec.streams, spec.logit_cap, spec.post_norms) == (3, 12.0, False)
    a, l, s = spec.layers[1].mixer, spec.layers[2].mixer, spec.layers[0].mixer
    assert (a.window, a.chunk, a.sink, a.bias, a.qk_norm, a.rotary) == (17, 0, True, False, False, None)
    assert (l.rank, l.rotary) == (72, RotarySpec(8, 700.0)) and (s.channels, s.state, s.dt_rank, s.taps) == (88, 24, 8, 4)
    assert spec.layers[2].mlp is None and spec.layers[0].mlp.activation == "relu2"
    assert roletar_spec(CONFIGS["roletar_many"]).layers[1].mixer.window == 0
    for bad in (layer(WIN, kv_heads=4), layer(LATENT, rot=dict(base=10.0, dims=4)), dict(WIN, type="gla"),
                dict(WIN, mlp=dict(kind="moe", ff=8))):
        with pytest.raises(ValueError):
            roletar_spec(roletar([bad]))
    with pytest.raises(ValueError):          # what streams do not go with
        DecoderSpec(vocab=8, width=8, eps=0.1, layers=(), streams=2)
    w = random_weights(cfg)
    w["l3.norm2"], w["l3.hc2.in"] = torch.ones(72), torch.ones(3)      # of a feed-forward that layer 3 does not have
    write_checkpoint(tmp_path, cfg, w)
    m = model_from_config(str(tmp_path), dtype=torch.float32)
    into, out_of = m.layers[2].mixer.per_head()
    uk, uv = w["l2.mix.uk"].float(), w["l2.mix.uv"].float()
    assert torch.equal(into[3], uk[3 * 24:4 * 24].T) and torch.equal(out_of[4], uv[4 * 40:])
    assert len(m.layers[0].linears()) == 5 and len(m.layers[2].linears()) == 2
    del w["l1.mix.sink"]
    write_checkpoint(tmp_path, cfg, w)
    with pytest.raises(ValueError):
        model_from_config(str(tmp_path))


def test_cache_rows_of_latents():
    from nanoquantization_amd.engine.hybrid_ops import latent_row
    bf, fp = torch.bfloat16, torch.float32
    assert latent_row(512, 64, bf) == (512, 576) and latent_row(50, 6, bf) == (64, 96) and latent_row(65, 33, bf) == (128, 192)
    assert latent_row(50, 6, fp) == (50, 56) and latent_row(600, 64, bf) == (600, 664) and latent_row(64, 80, bf) == (64, 144)


def test_registry_picks_by_config(tmp_path):
    assert registry.find_architecture({"architecture": "Roletar"}).step_kernels == "hybrid"
    assert registry.find_architecture({"architecture": "Gafulix"}).name == "Gafulix"
    assert registry.find_architecture({"quantization_config": {}}).name == "Qwen3Quantized"
    with pytest.raises(ValueError):
        registry.find_architecture({"architecture": "Unheard"})
    from nanoquantization_amd.engine import HybridEngine, LLMEngine
    m = GafulixForCausalLM(spec_from_config(CONFIGS["no_loop"]))
    assert registry.engine_for(m) is HybridEngine and registry.engine_for(torch.nn.Module()) is LLMEngine
    with pytest.raises(RuntimeError):          # no CPU path
        HybridEngine(m, 1, 16)


def test_spec_validation_and_runs():
    spec = spec_from_config(CONFIGS["loop_middle"])
    assert spec.runs() == o.layer_schedule(CONFIGS["loop_middle"]) == [
        (0, False), (1, False), (2, False), (1, True), (2, False), (1, True), (2, False), (3, False)]
    assert spec_from_config(CONFIGS["loop_all"]).runs() == [(0, False), (1, False), (0, True), (1, False)]
    assert spec_from_config(CONFIGS["one_pass_loop"]).runs() == [(0, False), (1, False)]
    with pytest.raises(ValueError):
        spec_from_config(config([layer(ATT, kv_heads=4)]))
    with pytest.raises(ValueError):
        spec_from_config(config([layer(ATT)], dict(start=0, stop=2, times=2)))
    with pytest.raises(ValueError):
        spec_from_config(config([dict(ATT, type="other")]))


@pytest.mark.parametrize("dims,base,scaling", [
    (24, 500.0, dict(factor=3.0, original=64, fast=8.0, slow=0.5)), (96, 10000.0, None),
    (64, 10000.0, dict(factor=8.0, original=4096, fast=32.0, slow=1.0)),
    (16, 100.0, dict(factor=2.0, original=8, fast=64.0, slow=32.0))])       # both ends clamp to the same pair
def test_rotary_table_against_plain_formula(dims, base, scaling):
    sc = YarnScaling(scaling["factor"], scaling["original"], scaling["fast"], scaling["slow"]) if scaling else None
    table = rotary_table(RotarySpec(dims, base, sc), 200)
    assert table.shape == (200, dims) and table.dtype == torch.float32
    freqs, mag = o.rotary_frequencies(dims, base, scaling)
    f = torch.tensor(freqs, dtype=torch.float64)
    for p in (0, 1, 63, 199):
        assert torch.allclose(table[p].double(), torch.cat([(p * f).cos(), (p * f).sin()]) * mag, atol=1e-6)
    if scaling:
        plain, _ = o.rotary_frequencies(dims, base)
        assert freqs[0] in (plain[0], plain[0] / scaling["factor"]) and abs(freqs[-1] - plain[-1]) <= plain[-1]


def test_caches_hand_out_and_take_back():
    c = PagedKVCache(3, 5, 4, dtype=torch.float32, device="cpu", layer_shapes=[(2, 32, 64), None, (1, 8, 8)])
    assert c.k[0].shape == (5, 2, 4, 32) and c.v[0].shape == (5, 2, 4, 64) and c.k[1] is None and c.v[2].shape == (5, 1, 4, 8)
    a = c.allocate(3)
    with pytest.raises(RuntimeError):
        c.allocate(3)
    c.release(a)
    assert sorted(c.free) == list(range(5))
    s = RecurrentStateCache(2, [None, (3, 4, 5)], "cpu")
    assert s.state[0] is None and s.state[1].shape == (2, 3, 4, 5) and s.state[1].dtype == torch.float32
    t = RecurrentStateCache(3, [(2, 6), None], "cpu", [(4, 6), None])
    assert t.tail[0].shape == (3, 4, 6) and t.tail[1] is None and s.tail == [None, None]
    x, y = s.allocate(), s.allocate()
    assert {x, y} == {0, 1}
    with pytest.raises(RuntimeError):
        s.allocate()
    s.release(x)
    assert s.allocate() == x


def test_oracle_mechanisms_consistent():
    """Closed forms: a recurrence written out as a sum, a chunked mask as separate sequences, a loop as copied layers."""
    g = torch.Generator().manual_seed(0)
    q, k = torch.randn(9, 2, 5, generator=g).double(), torch.randn(9, 2, 5, generator=g).double()
    v, a = torch.randn(9, 2, 3, generator=g).double(), torch.rand(9, 2, 5, generator=g).double()
    out, S = o.gla_scan(q, k, v, a)
    t = 7
    want = sum(((q[t] * k[j] * a[j + 1:t + 1].prod(dim=0)).sum(-1, keepdim=True) * v[j]) for j in range(t + 1))
    assert torch.allclose(out[t], want)
    o1, s1 = o.gla_scan(q[:4], k[:4], v[:4], a[:4])
    o2, s2 = o.gla_scan(q[4:], k[4:], v[4:], a[4:], s1)
    assert torch.allclose(torch.cat([o1, o2]), out) and torch.allclose(s2, S)
    whole = o.attend(q, k, v, 0.7, chunk=4)
    parts = torch.cat([o.attend(q[i:i + 4], k[i:i + 4], v[i:i + 4], 0.7) for i in range(0, 9, 4)])
    assert torch.allclose(whole, parts)
    # a window as a matrix, a sink as a further key that scores it and has no value
    s = torch.einsum("ihd,jhd->hij", q, k) * 0.7
    i, j = torch.arange(9).view(9, 1), torch.arange(9)
    s = s.masked_fill(~((j <= i) & (i - j < 4)), -torch.inf)
    sink = torch.tensor([0.3, 5.0]).double()
    p = torch.softmax(torch.cat([s, sink.view(2, 1, 1).expand(2, 9, 1)], -1), -1)[..., :9]
    assert torch.allclose(o.attend(q, k, v, 0.7, window=4, sink=sink), torch.einsum("hij,jhd->ihd", p, v))
    # latent attention as plain attention over expanded keys that repeat the shared part
    wl = {n: torch.randn(*sh, generator=g).double() for n, sh in dict(q=(2 * 7, 6), dkv=(5 + 4, 6), uk=(2 * 3, 5), uv=(2 * 4, 5),
                                                                      o=(6, 8)).items()}
    wl["dkv.norm"] = torch.rand(5, generator=g).double()
    h = torch.randn(4, 6, generator=g).double()
    got = o.latent_attention_mixer(h, wl, dict(heads=2, dim=3, rot_dim=4, vdim=4, kv_rank=5, scale=0.4, rot=dict(base=9.0)), 1e-3)
    down = h @ wl["dkv"].T
    c = o.rms(down[:, :5], wl["dkv.norm"], 1e-3)
    z = torch.polar(torch.ones(4, 2).double(), torch.arange(4).view(4, 1) * torch.tensor([1.0, 1 / 3]).double())
    turn = lambda x: torch.view_as_real(torch.view_as_complex(x.reshape(4, -1, 2, 2).contiguous()) * z.unsqueeze(1)).reshape(4, -1, 4)
    qq = (h @ wl["q"].T).view(4, 2, 7)
    kk = torch.cat([(c @ wl["uk"].T).view(4, 2, 3), turn(down[:, 5:]).expand(4, 2, 4)], -1)
    s = torch.einsum("ihd,jhd->hij", torch.cat([qq[..., :3], turn(qq[..., 3:])], -1), kk) * 0.4
    p = torch.softmax(s.masked_fill(j[:4] > i[:4], -torch.inf), -1)
    assert torch.allclose(got, torch.einsum("hij,jhd->ihd", p, (c @ wl["uv"].T).view(4, 2, 4)).reshape(4, 8) @ wl["o"].T)
    # the scan written out as a sum, and cut in two
    x, dt, A = torch.randn(6, 3, generator=g).double(), torch.rand(6, 3, generator=g).double(), -torch.rand(3, 4, generator=g).double()
    B, C, D = torch.randn(6, 4, generator=g).double(), torch.randn(6, 4, generator=g).double(), torch.randn(3, generator=g).double()
    y, S = o.selective_scan(x, dt, A, B, C, D)
    want = sum((torch.exp(dt[u + 1:6].sum(0)[:, None] * A) * (dt[u] * x[u])[:, None] * B[u]) @ C[5] for u in range(6)) + D * x[5]
    assert torch.allclose(y[5], want)
    y1, S1 = o.selective_scan(x[:2], dt[:2], A, B[:2], C[:2], D)
    y2, S2 = o.selective_scan(x[2:], dt[2:], A, B[2:], C[2:], D, S1)
    assert torch.allclose(torch.cat([y1, y2]), y) and torch.allclose(S2, S)
    wc, bc = torch.randn(3, 4, generator=g).double(), torch.randn(3, generator=g).double()
    conv = o.short_conv(x, wc, bc)
    assert torch.allclose(conv[1], wc[:, 3] * x[1] + wc[:, 2] * x[0] + bc)
    assert torch.allclose(o.short_conv(x[3:], wc, bc, x[:3]), conv[3:])
    # hyper-connections that only add are the plain residual
    xs = torch.stack([x, x * 0])
    new = o.hyper_write(xs, torch.tensor([[1.0, 0.5], [0.0, 1.0]]).double(), torch.tensor([1.0, 0.0]).double(), dt)
    assert torch.allclose(new[0], x + dt) and torch.allclose(new[1], 0.5 * x)
    cfg = CONFIGS["one_pass_loop"]
    w = random_weights(cfg)
    ids = tokens(6, cfg["vocab"])
    assert torch.allclose(o.gafulix_logits(cfg, w, ids), o.gafulix_logits(dict(cfg, loop=None), w, ids))
    # the weight is inside the expert: not the same as scaling its output
    w2 = {"router": torch.randn(3, 4, generator=g).double()}
    for e in range(3):
        w2[f"e{e}.gate"], w2[f"e{e}.up"] = torch.randn(6, 4, generator=g).double(), torch.randn(6, 4, generator=g).double()
        w2[f"e{e}.down"] = torch.randn(4, 6, generator=g).double()
    h = torch.randn(2, 4, generator=g).double()
    y = o.moe(h, w2, dict(router=dict(top=1)))
    (e, s), = o.route(h, w2["router"], 1)[0]
    inside = w2[f"e{e}.down"] @ (o.silu(w2[f"e{e}.gate"] @ h[0] * s) * (w2[f"e{e}.up"] @ h[0] * s))
    assert torch.allclose(y[0], inside)
