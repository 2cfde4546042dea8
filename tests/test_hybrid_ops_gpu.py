"""Kernels of the hybrid decoders against the plain oracle, each mechanism alone, in bf16 and in fp32."""
import pytest
import torch

from nanoquantization_amd import _lib
from nanoquantization_amd.engine import hybrid_ops as ops
from oracle import hybrid_oracle as o

pytestmark = pytest.mark.gpu
DTYPES = [torch.float32, torch.bfloat16]
TOL = {torch.float32: 2e-5, torch.bfloat16: 1.5e-2}


def rand(*shape, seed=0, dtype=torch.float32, scale=1.0):
    g = torch.Generator().manual_seed(seed)
    return (torch.randn(*shape, generator=g) * scale).to(dtype)


def close(got, want, dtype, what=""):
    got, want = got.double().cpu(), want.double()
    assert got.shape == want.shape, (what, got.shape, want.shape)
    err, ref = (got - want).abs().max().item(), want.abs().max().item()
    assert err <= TOL[dtype] * max(ref, 1e-3), (what, dtype, err, ref)


# ---- the step between two sublayers ----------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows,width,parts", [(3, 72, 1), (5, 1024, 3), (2, 8192, 2), (4, 50, 2), (1, 7, 1)])
def test_residual_norm(dtype, rows, width, parts):
    print(f"residual_norm {rows}x{width} parts={parts} {dtype}", flush=True)
    x0, y = rand(rows, width, seed=1), rand(rows, parts, width, seed=2, dtype=dtype)
    wb, wn = rand(width, seed=3, dtype=dtype), rand(width, seed=4, dtype=dtype)
    table, ids = rand(9, width, seed=5, dtype=dtype), torch.tensor([i % 9 for i in range(rows)])
    c = lambda t: t.cuda().contiguous()
    eps = 1e-3
    # everything at once
    x = c(x0)
    h = ops.residual_norm(x, eps, y=c(y), post_weight=c(wb), ids=c(ids), table=c(table), next_weight=c(wn))
    want = x0.double() + o.rms(y.double().sum(1), wb.double(), eps) + table.double()[ids]
    close(x, want, torch.float32, "x")
    close(h, o.rms(want, wn.double(), eps), dtype, "h")
    # start of a pass over the layers
    x = torch.full((rows, width), float("nan"), device="cuda")
    h = ops.residual_norm(x, eps, init=True, ids=c(ids), table=c(table), next_weight=c(wn))
    close(x, table.double()[ids], torch.float32)
    close(h, o.rms(table.double()[ids], wn.double(), eps), dtype)
    # addition without a norm of its own, no successor
    x = c(x0)
    assert ops.residual_norm(x, eps, y=c(y)) is None
    close(x, x0.double() + y.double().sum(1), torch.float32)


# ---- q/k norm, rotary, cache write --------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,dim,vdim,rot,norm", [(6, 2, 40, 24, 24, True), (4, 4, 64, 64, 64, True), (3, 1, 22, 26, 10, True),
                                                  (4, 2, 128, 96, 0, True), (8, 2, 32, 48, 32, False)])
def test_qk_norm_rope_store(dtype, H, G, dim, vdim, rot, norm):
    print(f"qk_norm_rope_store H={H} G={G} dim={dim} vdim={vdim} rot={rot} {dtype}", flush=True)
    rows, bs, blocks, eps, base = 5, 4, 6, 1e-4, 300.0
    kr, vr = ((dim + 31) // 32 * 32, (vdim + 31) // 32 * 32) if dtype == torch.bfloat16 else (dim, vdim)
    qkv = rand(rows, H * dim + G * (dim + vdim), seed=1, dtype=dtype)
    qw, kw = rand(H * dim, seed=2, dtype=dtype), rand(G * dim, seed=3, dtype=dtype)
    pos = torch.tensor([0, 3, 17, 40, 41])
    slots = torch.tensor([5, 23, -1, 0, 10])
    freqs, mag = o.rotary_frequencies(rot, base, dict(factor=2.0, original=32, fast=4.0, slow=0.5)) if rot else ([], 1.0)
    table = None
    if rot:
        ang = torch.arange(64, dtype=torch.float64).unsqueeze(1) * torch.tensor(freqs, dtype=torch.float64)
        table = torch.cat([ang.cos() * mag, ang.sin() * mag], 1).float().cuda()
    kc = torch.zeros(blocks, G, bs, kr, dtype=dtype, device="cuda")
    vc = torch.zeros(blocks, G, bs, vr, dtype=dtype, device="cuda")
    q = ops.qk_norm_rope_store(qkv.cuda(), qw.cuda() if norm else None, kw.cuda() if norm else None, table, pos.cuda(),
                               slots.cuda(), kc, vc, H, dim, vdim, eps)
    d = qkv.double()
    wq, wk = d[:, :H * dim], d[:, H * dim:(H + G) * dim]
    if norm:
        wq, wk = o.rms(wq, qw.double(), eps), o.rms(wk, kw.double(), eps)
    wq, wk = wq.reshape(rows, H, dim), wk.reshape(rows, G, dim)
    if rot:
        wq = torch.stack([o.rotate_interleaved(wq[t], int(pos[t]), freqs, mag, rot) for t in range(rows)])
        wk = torch.stack([o.rotate_interleaved(wk[t], int(pos[t]), freqs, mag, rot) for t in range(rows)])
    close(q[..., :dim], wq, dtype, "q")
    assert torch.count_nonzero(q[..., dim:]) == 0
    wv = d[:, (H + G) * dim:].reshape(rows, G, vdim)
    ek, ev = torch.zeros(kc.shape, dtype=torch.float64), torch.zeros(vc.shape, dtype=torch.float64)
    for t, s in enumerate(slots.tolist()):
        if s >= 0:
            ek[s // bs, :, s % bs, :dim], ev[s // bs, :, s % bs, :vdim] = wk[t], wv[t]
    close(kc, ek, dtype, "k")
    close(vc, ev, dtype, "v")


# ---- attention ----------------------------------------------------------------------------------------------------
def paged(k, v, bs, dtype, spare=3, seed=9):
    """One sequence's keys and values [T, G, d] scattered over cache blocks; unused rows hold garbage."""
    T, G, dim = k.shape
    vdim = v.shape[2]
    kr, vr = ops.cache_rows(dim, vdim, dtype)
    nb = -(-T // bs)
    table = torch.randperm(nb + spare, generator=torch.Generator().manual_seed(seed))[:nb]
    kc = torch.full((nb + spare, G, bs, kr), 1e4, dtype=dtype)
    vc = torch.full((nb + spare, G, bs, vr), 1e4, dtype=dtype)
    kc[..., dim:], vc[..., vdim:] = 0, 0
    for t in range(T):
        b, i = int(table[t // bs]), t % bs
        kc[b, :, i, :dim], vc[b, :, i, :vdim] = k[t].to(dtype), v[t].to(dtype)
    return kc.cuda(), vc.cuda(), table.to(torch.int32).cuda()


def span(start, rows, table, bs):
    """The pass of one portion of the sequence whose block table is `table`."""
    return ops.PromptPass([(start, rows, table.tolist(), 0)], bs, torch.device("cuda"))


def padded_q(q, width, dtype):
    out = torch.zeros(q.shape[0], q.shape[1], width, dtype=dtype)
    out[..., :q.shape[2]] = q.to(dtype)
    return out.cuda()


ATTENTION = [  # T, H, G, dim, vdim, block, chunk
    (70, 4, 2, 40, 24, 16, 20), (130, 2, 1, 64, 64, 32, 0), (150, 3, 3, 96, 96, 64, 48), (65, 6, 1, 32, 48, 16, 7),
    (200, 4, 2, 128, 128, 64, 128), (100, 8, 1, 128, 64, 16, 64), (90, 2, 1, 192, 160, 32, 33), (80, 2, 2, 256, 256, 64, 0),
    (140, 16, 1, 64, 96, 16, 100), (75, 40, 2, 32, 32, 16, 50), (40, 2, 2, 22, 18, 16, 5), (33, 1, 1, 16, 16, 16, 1), (600, 2, 1, 64, 64, 64, 512)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,H,G,dim,vdim,bs,chunk", ATTENTION)
def test_attention_prefill_portions_and_decode(dtype, T, H, G, dim, vdim, bs, chunk):
    print(f"attention T={T} H={H} G={G} dim={dim} vdim={vdim} bs={bs} chunk={chunk} {dtype}", flush=True)
    q, k, v = (rand(T, H, dim, seed=1, dtype=dtype), rand(T, G, dim, seed=2, dtype=dtype), rand(T, G, vdim, seed=3, dtype=dtype))
    scale = dim ** -0.5 * 1.7
    want = o.attend(q.double(), k.double(), v.double(), scale, chunk).reshape(T, H * vdim)
    kc, vc, table = paged(k, v, bs, dtype)
    qd = padded_q(q, kc.shape[3], dtype)
    close(ops.attention_prefill(qd, kc, vc, span(0, T, table, bs), dim, vdim, scale, chunk), want, dtype, "whole")
    at = 0
    for n in (2, 3, 17, 16, 1, 31, T):      # portions that start and end anywhere
        n = min(n, T - at)
        if n:
            got = ops.attention_prefill(qd[at:at + n].contiguous(), kc, vc, span(at, n, table, bs), dim, vdim, scale, chunk)
            close(got, want[at:at + n], dtype, f"portion {at}+{n}")
        at += n
    # decode: every position at once, one row each
    rows = torch.tensor(sorted({0, 1, T // 2, T - 1, T - 2} | {c for e in range(0, T, max(chunk, 16)) for c in (e - 1, e, e + 1)
                                                           if 0 <= c < T}))
    tables = table.repeat(len(rows), 1).contiguous()
    got = ops.attention_decode(qd[rows.cuda()].contiguous(), kc, vc, tables, (rows + 1).to(torch.int32).cuda(), dim, vdim,
                               scale, chunk)
    close(got, want[rows], dtype, "decode")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("chunk,bs", [(48, 16), (50, 16), (0, 32), (300, 64)])
def test_attention_one_key_stands_out(dtype, chunk, bs):
    """A key that only one query points at, placed at the chunk's first token, just before it, at block borders and far
    away: the output must be that key's value exactly when the mask lets it through."""
    T, dim = 400, 64
    print(f"attention needle chunk={chunk} bs={bs} {dtype}", flush=True)
    for i in (399, 349, 200, 150):
        first = i // chunk * chunk if chunk else 0
        spots = {first, first + 1, first - 1, i, i - 1, i // bs * bs, i // bs * bs - 1, first + (i - first) // 2, 0}
        for j in sorted(s for s in spots if 0 <= s <= i):
            k, v = rand(T, 1, dim, seed=4, scale=0.1), rand(T, 1, dim, seed=5)
            q = rand(T, 1, dim, seed=6, scale=0.1)
            e = torch.zeros(dim)
            e[7] = 20.0
            q[i, 0], k[j, 0] = e, e
            kc, vc, table = paged(k, v, bs, dtype)
            qd = padded_q(q, dim, dtype)
            seen = o.visible(i, j, chunk)
            # alone, from a portion cut right in front of it, and decoded
            outs = [ops.attention_prefill(qd[i:i + 1].contiguous(), kc, vc, span(i, 1, table, bs), dim, dim, 0.125, chunk)[0],
                    ops.attention_prefill(qd[max(0, i - 40):i + 1].contiguous(), kc, vc,
                                          span(max(0, i - 40), min(i, 40) + 1, table, bs), dim, dim, 0.125, chunk)[-1],
                    ops.attention_decode(qd[i:i + 1].contiguous(), kc, vc, table.unsqueeze(0).contiguous(),
                                         torch.tensor([i + 1], dtype=torch.int32).cuda(), dim, dim, 0.125, chunk)[0]]
            for n, got in enumerate(outs):
                diff = (got.float().cpu() - v[j, 0]).abs().max().item()
                assert (diff < 2e-2) == seen, (i, j, chunk, n, diff, seen)


def test_attention_decode_long_context():
    """Contexts long enough for the context split, ragged over the batch."""
    dtype, T, G, H, dim, bs = torch.bfloat16, 3000, 2, 8, 64, 64
    k, v = rand(T, G, dim, seed=1, dtype=dtype), rand(T, G, dim, seed=2, dtype=dtype)
    kc, vc, table = paged(k, v, bs, dtype)
    ctx = torch.tensor([3000, 2999, 1, 65, 2049, 700], dtype=torch.int32)
    q = rand(len(ctx), H, dim, seed=3, dtype=dtype)
    for chunk in (0, 2048, 100):
        print(f"long decode chunk={chunk}", flush=True)
        got = ops.attention_decode(q.cuda(), kc, vc, table.repeat(len(ctx), 1).contiguous(), ctx.cuda(), dim, dim, 0.2, chunk)
        for b, n in enumerate(ctx.tolist()):
            lo = (n - 1) // chunk * chunk if chunk else 0
            kk, vv = k[lo:n].double(), v[lo:n].double()
            for h in range(H):
                s = kk[:, h // 4] @ q[b, h].double() * 0.2
                close(got[b, h * dim:(h + 1) * dim], torch.softmax(s, 0) @ vv[:, h // 4], dtype, (chunk, b, h))


# ---- gated linear attention ------------------------------------------------------------------------------------------
GLA_CASES = [(1, 2, 24, 40), (37, 3, 24, 40), (64, 2, 64, 64), (150, 2, 32, 32), (130, 1, 128, 128), (100, 2, 96, 48),
             (70, 1, 256, 256), (45, 2, 20, 12), (700, 1, 64, 96)]


def gla_inputs(T, H, dim, vdim, rank, dtype, seed=0, zshift=2.0):
    proj = rand(T, 2 * H * dim + 2 * H * vdim + rank, seed=seed, dtype=dtype)
    up = rand(H * dim, rank, seed=seed + 1, dtype=dtype, scale=rank ** -0.5)
    bias = (rand(H * dim, seed=seed + 2) + zshift).to(dtype)
    norm = (1 + 0.3 * rand(vdim, seed=seed + 3)).to(dtype)
    return proj, up, bias, norm


def gla_want(proj, up, bias, H, dim, vdim, tau, state=None):
    T = proj.shape[0]
    d = proj.double()
    q, k, v, g, low = d.split([H * dim, H * dim, H * vdim, H * vdim, up.shape[1]], dim=1)
    decay = o.channel_decay(low @ up.double().T + bias.double(), tau).view(T, H, dim)
    out, S = o.gla_scan(q.view(T, H, dim) * dim ** -0.5, k.view(T, H, dim), v.view(T, H, vdim), decay, state)
    return out, S, decay, g


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,H,dim,vdim", GLA_CASES)
@pytest.mark.parametrize("tau,zshift", [(4.0, 2.0), (1.0, -6.0)])
def test_gla_prefill_portions_and_decode(dtype, T, H, dim, vdim, tau, zshift):
    """zshift -6 at tau 1: decays of e^-6 and below a token, where a factored form of the decay would overflow."""
    rank, slots, eps = 10, 3, 1e-4
    print(f"gla T={T} H={H} dim={dim} vdim={vdim} tau={tau} {dtype}", flush=True)
    proj, up, bias, norm = gla_inputs(T, H, dim, vdim, rank, dtype, zshift=zshift)
    want, S, decay, g = gla_want(proj, up, bias, H, dim, vdim, tau)
    pd, ud, bd = proj.cuda(), up.cuda(), bias.cuda()
    dec = ops.gla_decay(pd, ud, bd, H, dim, vdim, tau)
    close(dec, decay.reshape(T, -1), torch.float32, "decay")
    # fp32 arithmetic on the given operands in either type: the tolerance is fp32's
    for cuts in ([T], [2] * (T // 2) + [T % 2], [T // 3, 16, T]):
        state = torch.full((slots, H, dim, vdim), 1e3, device="cuda")       # a slot is taken over as it is
        out = torch.empty(T, H * vdim, device="cuda")
        at = 0
        for n in cuts:
            n = min(n, T - at)
            if n > 0:
                one = ops.PromptPass([(at, n, range(T), 1)], 1, torch.device("cuda"))
                out[at:at + n] = ops.gla_prefill(pd[at:at + n], dec[at:at + n], state, one, H, dim, vdim, rank)
                at += n
        assert at == T
        close(out, want.reshape(T, -1), torch.float32, f"o {cuts[:2]}")
        close(state[1], S, torch.float32, "state")
        assert (state[0] == 1e3).all() and (state[2] == 1e3).all()
    gated = ops.head_norm_gate(out, pd, norm.cuda(), H, dim, vdim, rank, eps)
    wg = o.rms(want, norm.double(), eps).reshape(T, -1) * o.silu(g)
    close(gated, wg, dtype, "gated")
    # token by token, an idle row and a foreign slot beside it
    state = torch.full((slots, H, dim, vdim), 1e3, device="cuda")
    active = torch.tensor([True, False], device="cuda")
    slot = torch.tensor([2, 0], dtype=torch.int32, device="cuda")
    steps = min(T, 40)
    for t in range(steps):
        got = ops.gla_decode(pd[t:t + 1].repeat(2, 1), ud, bd, norm.cuda(), state, slot,
                             torch.tensor([t, t], device="cuda"), active, H, dim, vdim, tau, eps)
        close(got[0], wg[t], dtype, f"decode {t}")
        assert torch.count_nonzero(got[1]) == 0
    close(state[2], gla_want(proj[:steps], up, bias, H, dim, vdim, tau)[1], torch.float32, "decode state")
    assert (state[0] == 1e3).all() and (state[1] == 1e3).all()


@pytest.mark.parametrize("T", [300, 2100])
def test_gla_remembers_one_far_token(T):
    """Decays near 1 and one large key/value at the start, in the middle, at piece borders: the last token reads it."""
    H, dim, vdim, rank = 1, 32, 32, 4
    for j in (0, 15, 16, 63, 64, 255, 256, T - 1):
        print(f"gla needle T={T} j={j}", flush=True)
        proj = rand(T, 2 * dim + 2 * vdim + rank, seed=3, scale=0.01)
        proj[j, dim + 5] = proj[T - 1, 5] = 30.0
        up, bias = rand(dim, rank, seed=1), torch.full((dim,), 9.0)
        pd = proj.cuda()
        dec = ops.gla_decay(pd, up.cuda(), bias.cuda(), H, dim, vdim, 16.0)
        state = torch.zeros(1, H, dim, vdim, device="cuda")
        out = ops.gla_prefill(pd, dec, state, ops.PromptPass([(0, T, range(T), 0)], 1, torch.device("cuda")), H, dim, vdim, rank)
        q, k, v, _, _ = proj.double().split([dim, dim, vdim, vdim, rank], dim=1)
        d = dec.double().cpu()
        w = torch.cat([torch.flip(torch.cumprod(torch.flip(d[1:], [0]), 0), [0]), torch.ones(1, dim).double()])
        want = ((q[T - 1] * dim ** -0.5 * w * k).sum(-1, keepdim=True) * v).sum(0)
        close(out[T - 1], want, torch.float32, j)


@pytest.mark.parametrize("dtype", DTYPES)
def test_ragged_pass_equals_each_sequence_alone(dtype):
    """Portions of several sequences, some in their middle, long enough for several pieces and tiles, in one launch."""
    H, G, dim, vdim, bs, chunk, rank = 4, 2, 64, 48, 16, 100, 8
    portions = [(0, 300), (37, 150), (0, 1), (250, 2), (128, 128)]           # (start, rows)
    total = [s + n for s, n in portions]
    kr, vr = ops.cache_rows(dim, vdim, dtype)
    nb = [-(-t // bs) for t in total]
    order = torch.randperm(sum(nb), generator=torch.Generator().manual_seed(2)).tolist()
    kc, vc = (rand(sum(nb), G, bs, w, seed=7 + w, dtype=dtype).cuda() for w in (kr, vr + 0))
    blocks = [[order.pop() for _ in range(n)] for n in nb]
    segs = [(s, n, b, i) for i, ((s, n), b) in enumerate(zip(portions, blocks))]
    q = rand(sum(n for _, n in portions), H, kr, seed=3, dtype=dtype).cuda()
    print(f"ragged pass {dtype}", flush=True)
    dev = torch.device("cuda")
    got = ops.attention_prefill(q, kc, vc, ops.PromptPass(segs, bs, dev), dim, vdim, 0.1, chunk)
    HG, dg, vg = 16, 64, 80
    proj, up, bias, _ = gla_inputs(q.shape[0], HG, dg, vg, rank, dtype)
    proj, dec = proj.cuda(), None
    dec = ops.gla_decay(proj, up.cuda(), bias.cuda(), HG, dg, vg, 8.0)
    s0 = rand(len(segs), HG, dg, vg, seed=5).cuda()
    state = s0.clone()
    layout = ops.PromptPass(segs, bs, dev)
    assert layout.pieces(_lib.hybrid_lib().nqh_gla_piece_rows(q.shape[0], HG, dg, vg))[2]     # a sequence of several pieces
    o = ops.gla_prefill(proj, dec, state, layout, HG, dg, vg, rank)
    at = 0
    for i, seg in enumerate(segs):
        n = seg[1]
        one = ops.PromptPass([seg], bs, dev)
        alone = ops.attention_prefill(q[at:at + n].contiguous(), kc, vc, one, dim, vdim, 0.1, chunk)
        close(got[at:at + n], alone.double().cpu(), dtype, i)
        st = s0.clone()
        oi = ops.gla_prefill(proj[at:at + n].contiguous(), dec[at:at + n].contiguous(), st, one, HG, dg, vg, rank)
        close(o[at:at + n], oi.double().cpu(), torch.float32, i)
        close(state[i], st[i].double().cpu(), torch.float32, i)
        at += n


# ---- mixture of experts --------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows,width,experts,top,ff", [(1, 72, 5, 2, 48), (37, 64, 9, 1, 40), (20, 128, 7, 7, 64),
                                                      (300, 96, 4, 2, 36), (3, 50, 3, 1, 21), (64, 256, 64, 6, 128), (5, 64, 200, 3, 32), (90, 96, 300, 4, 16), (6, 80, 1, 1, 24),
                                                      (1500, 128, 6, 2, 160), (700, 256, 3, 1, 96),
                                                      (40, 264, 4, 2, 72), (100, 128, 8, 2, 64), (120, 136, 4, 1, 200)])
def test_router_and_experts(dtype, rows, width, experts, top, ff):
    print(f"moe rows={rows} width={width} experts={experts} top={top} ff={ff} {dtype}", flush=True)
    h = rand(rows, width, seed=1, dtype=dtype)
    router = rand(experts, width, seed=2, dtype=dtype, scale=2 * width ** -0.5)
    gu, dn = rand(experts, 2 * ff, width, seed=3, dtype=dtype, scale=width ** -0.5), rand(experts, width, ff, seed=4, dtype=dtype, scale=ff ** -0.5)
    expert, weight = ops.router_topk(h.cuda(), router.cuda(), top)
    s = torch.sigmoid(h.double() @ router.double().T)
    ws, we = s.topk(top, dim=1)
    close(weight, ws, torch.float32, "scores")
    gap = s.sort(dim=1, descending=True).values[:, :top + 1]
    clear = (gap[:, :-1] - gap[:, 1:]).min(dim=1).values > 1e-5 if experts > 1 else torch.ones(rows, dtype=torch.bool)
    assert torch.equal(expert.cpu().long()[clear], we[clear]) and clear.float().mean() > 0.8
    y = ops.moe_experts(h.cuda(), gu.cuda(), dn.cuda(), ops.route(h.cuda(), router.cuda(), top, ff))
    assert y.shape == (rows, top, width)
    e, w = expert.cpu().long(), weight.cpu().double()
    u = h.double().unsqueeze(1) * w.unsqueeze(-1)                              # [rows, top, width]
    want = torch.empty(rows, top, width, dtype=torch.float64)
    for x in range(experts):
        at = (e == x).nonzero(as_tuple=True)
        if len(at[0]):
            a, b = u[at] @ gu[x, :ff].double().T, u[at] @ gu[x, ff:].double().T
            want[at] = (o.silu(a) * b) @ dn[x].double().T
    close(y, want, dtype, "experts")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows,width,experts,top,ff", [(1, 72, 5, 2, 48), (16, 2048, 8, 2, 64), (64, 256, 64, 6, 128),
                                                      (200, 1028, 128, 8, 32), (33, 4096, 3, 3, 24), (300, 64, 8, 2, 32)])
def test_residual_norm_route_equals_separate_launches(dtype, rows, width, experts, top, ff):
    print(f"norm + route rows={rows} width={width} experts={experts} top={top} {dtype}", flush=True)
    x0, y = rand(rows, width, seed=1).cuda(), rand(rows, 2, width, seed=2, dtype=dtype).cuda()
    wb, wn = rand(width, seed=3, dtype=dtype).cuda(), rand(width, seed=4, dtype=dtype).cuda()
    router = rand(experts, width, seed=5, dtype=dtype, scale=2 * width ** -0.5).cuda()
    for again in range(3):                 # the arrival counter is left as it was found
        x1, x2 = x0.clone(), x0.clone()
        h1 = ops.residual_norm(x1, 1e-5, y=y, post_weight=wb, next_weight=wn)
        h2, r = ops.residual_norm_route(x2, 1e-5, router, top, ff, wn, y=y, post_weight=wb)
        assert torch.equal(x1, x2) and torch.equal(h1, h2)
        s = torch.sigmoid(h1.double() @ router.double().T).cpu()
        ws, we = s.topk(top, dim=1)
        close(r.weight, ws, torch.float32, "scores")
        gap = s.sort(dim=1, descending=True).values[:, :top + 1]
        clear = (gap[:, :-1] - gap[:, 1:]).min(dim=1).values > 1e-5
        assert torch.equal(r.expert.cpu().long()[clear], we[clear]) and clear.float().mean() > 0.8
        e, order, tiles = r.expert.cpu().reshape(-1), r.order.cpu().long(), r.tiles.cpu()
        n, seen = r.max_tiles, 0
        assert sorted(order.tolist()) == list(range(rows * top))
        for t in range(int(tiles[-1])):
            ex, first, count = int(tiles[t]), int(tiles[n + t]), int(tiles[2 * n + t])
            assert 1 <= count <= r.tile_rows and first == seen and (e[order[first:first + count]] == ex).all()
            seen += count
        assert seen == rows * top


def test_moe_plan_groups_every_pair_once():
    for pairs, experts, rows in ((1, 1, 16), (1000, 7, 16), (5000, 64, 128), (300, 1000, 32)):
        print(f"plan pairs={pairs} experts={experts}", flush=True)
        e = torch.randint(0, experts, (pairs, 1), generator=torch.Generator().manual_seed(pairs), dtype=torch.int32)
        e[: pairs // 3] = e[0]
        order, tiles = ops.moe_plan(e.cuda(), experts, rows)
        order, tiles = order.cpu().long(), tiles.cpu()
        n = (tiles.numel() - 1) // 3
        assert sorted(order.tolist()) == list(range(pairs))
        seen = 0
        for t in range(int(tiles[-1])):
            ex, first, count = int(tiles[t]), int(tiles[n + t]), int(tiles[2 * n + t])
            assert 1 <= count <= rows and (e[order[first:first + count], 0] == ex).all() and first == seen
            seen += count
        assert seen == pairs


# ---- dense products, sampling ----------------------------------------------------------------------------------------
@pytest.mark.parametrize("rows,n_out,n_in", [(1, 440, 200), (3, 50, 8), (16, 1000, 1024), (17, 96, 136), (33, 256, 512),
                                             (64, 640, 4096), (5, 16, 128), (48, 33, 72)])
def test_skinny_linear(rows, n_out, n_in):
    print(f"skinny {rows} x {n_in} -> {n_out}", flush=True)
    x, w = rand(rows, n_in, seed=1, dtype=torch.bfloat16), rand(n_out, n_in, seed=2, dtype=torch.bfloat16)
    b = rand(n_out, seed=3, dtype=torch.bfloat16)
    want = x.double() @ w.double().T
    close(ops.skinny_linear(x.cuda(), w.cuda(), out_f32=True), want, torch.float32)
    close(ops.skinny_linear(x.cuda(), w.cuda(), b.cuda(), out_f32=True), want + b.double(), torch.float32)
    close(ops.skinny_linear(x.cuda(), w.cuda(), b.cuda()), want + b.double(), torch.bfloat16)


def test_argmax_and_bookkeeping():
    for rows, vocab in ((1, 5), (3, 131), (4, 32000), (2, 4098)):
        x = rand(rows, vocab, seed=vocab)
        x[0, vocab - 1] = x[0, 1] = 99.0
        assert torch.equal(ops.argmax_rows(x.cuda()).cpu(), x.argmax(-1).where(torch.arange(rows) > 0, torch.tensor(1)))
    pos, act = torch.tensor([0, 5, 9]).cuda(), torch.tensor([True, True, False]).cuda()
    table = torch.tensor([[3, 1, 0], [2, 4, 0], [5, 5, 5]], dtype=torch.int32).cuda()
    slots, ctx = ops.decode_prepare(pos, act, table, 4)
    assert slots.tolist() == [12, 17, -1] and ctx.tolist() == [1, 6, 10]
    log, ids, step = torch.zeros(2, 3, dtype=torch.long).cuda(), torch.zeros(3, dtype=torch.long).cuda(), torch.zeros(1, dtype=torch.long).cuda()
    ops.decode_advance(torch.tensor([7, 8, 9]).cuda(), act, log, ids, pos, step)
    assert log.tolist() == [[7, 8, 9], [0, 0, 0]] and ids.tolist() == [7, 8, 9] and pos.tolist() == [1, 6, 9] and step.item() == 1


def test_argument_checks_raise():
    q = torch.zeros(4, 2, 32, dtype=torch.bfloat16, device="cuda")
    kc = torch.zeros(2, 1, 16, 32, dtype=torch.bfloat16, device="cuda")
    table = torch.tensor([0], dtype=torch.int32, device="cuda")
    with pytest.raises(_lib.AwqHipError):                  # positions past the block table
        ops.attention_prefill(q, kc, kc, span(13, 4, table, 16), 32, 32, 1.0)
    with pytest.raises(_lib.AwqHipError):
        ops.skinny_linear(torch.zeros(65, 32, dtype=torch.bfloat16, device="cuda"), torch.zeros(8, 32, dtype=torch.bfloat16, device="cuda"))
    with pytest.raises(_lib.AwqHipError):
        ops.router_topk(torch.zeros(1, 8, device="cuda"), torch.zeros(2, 8, device="cuda"), 3)
    with pytest.raises(_lib.AwqHipError):
        ops.argmax_rows(torch.zeros(1, 8))
