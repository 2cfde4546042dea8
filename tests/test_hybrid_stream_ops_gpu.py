"""Kernels of windows and sinks, latent attention, selective scans and hyper-connections against the plain oracle, each
mechanism alone, in bf16 and in fp32."""
import pytest
import torch

from nanoquantization_amd import _lib
from nanoquantization_amd.engine import hybrid_ops as ops
from nanoquantization_amd.models.hybrid import RotarySpec, rotary_table
from oracle import hybrid_oracle as o
from test_hybrid_ops_gpu import DTYPES, close, padded_q, paged, rand, span

pytestmark = pytest.mark.gpu
DEV = "cuda"


# ---- hyper-connections, activations ----------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows,streams,width", [(3, 2, 72), (1, 1, 50), (5, 3, 1024), (2, 4, 2052), (2, 8, 4100), (300, 2, 96),
                                                (2, 5, 7), (1, 6, 8192)])
def test_hyper_norm(dtype, rows, streams, width):
    print(f"hyper_norm {rows}x{streams}x{width} {dtype}", flush=True)
    x0, y = rand(rows, streams, width, seed=1), rand(rows, width, seed=2, dtype=dtype)
    mix, write, read = rand(streams, streams, seed=3, dtype=dtype), rand(streams, seed=4, dtype=dtype), rand(streams, seed=5, dtype=dtype)
    wn, table, ids = rand(width, seed=6, dtype=dtype), rand(9, width, seed=7, dtype=dtype), torch.tensor([(3 * i) % 9 for i in range(rows)])
    c, eps = (lambda t: t.cuda().contiguous()), 1e-3
    x = c(x0)
    h = ops.hyper_norm(x, eps, y=c(y), mix=c(mix), write=c(write), read=c(read), next_weight=c(wn))
    xs = o.hyper_write(x0.double().transpose(0, 1), mix.double(), write.double(), y.double())
    close(x, xs.transpose(0, 1), torch.float32, "x")
    close(h, o.rms(o.hyper_read(xs, read.double()), wn.double(), eps), dtype, "h")
    # the end: the plain sum is read; no sublayer output
    close(ops.hyper_norm(x, eps, next_weight=c(wn)), o.rms(xs.sum(0), wn.double(), eps), dtype, "sum")
    close(x, xs.transpose(0, 1), torch.float32, "x unchanged")
    assert ops.hyper_norm(x, eps, y=c(y), mix=c(mix), write=c(write)) is None
    close(x, o.hyper_write(xs, mix.double(), write.double(), y.double()).transpose(0, 1), torch.float32, "no reader")
    # the start, whatever the buffer held
    x = torch.full((rows, streams, width), float("nan"), device=DEV)
    h = ops.hyper_norm(x, eps, ids=c(ids), table=c(table), read=c(read), next_weight=c(wn))
    emb = table.double()[ids]
    close(x, emb.unsqueeze(1).expand(-1, streams, -1), torch.float32, "start")
    close(h, o.rms(emb * read.double().sum(), wn.double(), eps), dtype, "start h")


@pytest.mark.parametrize("dtype", DTYPES)
def test_activations(dtype):
    for n in (1, 24, 4099, 8192):
        print(f"activations {n} {dtype}", flush=True)
        x = rand(n, seed=n, dtype=dtype, scale=3.0)
        close(ops.activate_(x.cuda(), "relu2"), x.double().clamp(min=0) ** 2, dtype)
        close(ops.activate_((20 * x).cuda(), "softcap", 7.0), o.softcap((20 * x).double(), 7.0), dtype)
    for rows in (2, 30, 64):        # behind a product
        x, w, b = (rand(*s, seed=i, dtype=torch.bfloat16) for i, s in enumerate([(rows, 72), (50, 72), (50,)]))
        z = x.double() @ w.double().T + b.double()
        close(ops.skinny_linear(x.cuda(), w.cuda(), b.cuda(), activation="relu2"), z.clamp(min=0) ** 2, torch.bfloat16)
        close(ops.skinny_linear(x.cuda(), w.cuda(), b.cuda(), True, "softcap", 4.0), o.softcap(z, 4.0), torch.float32)
    with pytest.raises(_lib.AwqHipError):
        ops.activate_(torch.ones(4, device=DEV), "softcap", 0.0)


# ---- windows and sinks ------------------------------------------------------------------------------------------------
WINDOWS = [  # T, H, G, dim, vdim, block, window
    (70, 4, 2, 40, 24, 16, 20), (130, 2, 1, 64, 32, 32, 0), (150, 3, 3, 96, 96, 64, 48), (65, 6, 1, 32, 48, 16, 7),
    (300, 4, 2, 128, 128, 64, 129), (100, 40, 2, 16, 64, 16, 64), (90, 2, 1, 192, 160, 32, 33), (60, 2, 2, 22, 18, 16, 1),
    (600, 2, 1, 64, 64, 64, 513), (50, 2, 2, 256, 200, 16, 500)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,H,G,dim,vdim,bs,window", WINDOWS)
def test_window_and_sink_prefill_portions_and_decode(dtype, T, H, G, dim, vdim, bs, window):
    print(f"window T={T} H={H} G={G} dim={dim} vdim={vdim} bs={bs} window={window} {dtype}", flush=True)
    q, k, v = (rand(T, H, dim, seed=1, dtype=dtype), rand(T, G, dim, seed=2, dtype=dtype), rand(T, G, vdim, seed=3, dtype=dtype))
    sink = (3.0 * rand(H, seed=4)).to(dtype)           # from negligible to most of the weight
    scale = dim ** -0.5 * 1.7
    want = o.attend(q.double(), k.double(), v.double(), scale, window=window, sink=sink.double()).reshape(T, H * vdim)
    kc, vc, table = paged(k, v, bs, dtype)
    qd, args = padded_q(q, kc.shape[3], dtype), (dim, vdim, scale, 0, window, sink.cuda())
    close(ops.attention_prefill(qd, kc, vc, span(0, T, table, bs), *args), want, dtype, "whole")
    at = 0
    for n in (2, 3, 17, 16, 1, 31, T):
        n = min(n, T - at)
        if n:
            got = ops.attention_prefill(qd[at:at + n].contiguous(), kc, vc, span(at, n, table, bs), *args)
            close(got, want[at:at + n], dtype, f"portion {at}+{n}")
        at += n
    rows = torch.tensor(sorted({0, 1, T // 2, T - 1} | {i for i in (window - 2, window - 1, window, window + 1) if 0 <= i < T}))
    got = ops.attention_decode(qd[rows.cuda()].contiguous(), kc, vc, table.repeat(len(rows), 1).contiguous(),
                               (rows + 1).to(torch.int32).cuda(), *args)
    close(got, want[rows], dtype, "decode")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("window,bs", [(48, 16), (50, 16), (0, 32), (200, 64), (1, 16)])
def test_window_edge_key_stands_out(dtype, window, bs):
    """A key that only one query points at, just inside and just outside the window, at block borders and far away; and the
    same score as a sink, which takes the weight and gives nothing."""
    T, dim = 400, 64
    print(f"window needle {window} bs={bs} {dtype}", flush=True)
    for i in (399, 250, 200, 63):
        first = max(0, i - window + 1) if window else 0
        spots = {first, first + 1, first - 1, i, i - 1, i // bs * bs, i // bs * bs - 1, 0}
        for j in sorted(s for s in spots if 0 <= s <= i):
            k, v = rand(T, 1, dim, seed=4, scale=0.1), rand(T, 1, dim, seed=5)
            q, e = rand(T, 1, dim, seed=6, scale=0.1), torch.zeros(dim)
            e[7] = 20.0
            q[i, 0], k[j, 0] = e, e
            kc, vc, table = paged(k, v, bs, dtype)
            qd, seen = padded_q(q, dim, dtype), o.visible(i, j, window=window)
            for strong in (False, True):         # the needle scores 50; a sink of 60 takes everything
                sink = torch.tensor([60.0 if strong else 0.0], dtype=dtype, device=DEV)
                args = (dim, dim, 0.125, 0, window, sink)
                outs = [ops.attention_prefill(qd[i:i + 1].contiguous(), kc, vc, span(i, 1, table, bs), *args)[0],
                        ops.attention_prefill(qd[max(0, i - 40):i + 1].contiguous(), kc, vc,
                                              span(max(0, i - 40), min(i, 40) + 1, table, bs), *args)[-1],
                        ops.attention_decode(qd[i:i + 1].contiguous(), kc, vc, table.unsqueeze(0).contiguous(),
                                             torch.tensor([i + 1], dtype=torch.int32).cuda(), *args)[0]]
                for n, got in enumerate(outs):
                    got = got.float().cpu()
                    if strong:
                        assert got.abs().max() < 2e-2, (i, j, window, n)
                    else:
                        assert ((got - v[j, 0]).abs().max().item() < 2e-2) == seen, (i, j, window, n, seen)


def test_window_and_sink_decode_over_context_splits():
    dtype, T, G, H, dim, bs = torch.bfloat16, 3000, 2, 8, 64, 64
    k, v = rand(T, G, dim, seed=1, dtype=dtype), rand(T, G, dim, seed=2, dtype=dtype)
    kc, vc, table = paged(k, v, bs, dtype)
    ctx = torch.tensor([3000, 2999, 1, 65, 2049, 700], dtype=torch.int32)
    q, sink = rand(len(ctx), H, dim, seed=3, dtype=dtype), (2 * rand(H, seed=5) + 3).to(dtype)
    for window in (0, 2048, 1100, 100):
        print(f"long decode window={window}", flush=True)
        got = ops.attention_decode(q.cuda(), kc, vc, table.repeat(len(ctx), 1).contiguous(), ctx.cuda(), dim, dim, 0.2, 0,
                                   window, sink.cuda())
        for b, n in enumerate(ctx.tolist()):
            lo = max(0, n - window) if window else 0
            for h in range(H):
                s = torch.cat([k[lo:n, h // 4].double() @ q[b, h].double() * 0.2, sink[h:h + 1].double()])
                close(got[b, h * dim:(h + 1) * dim], torch.softmax(s, 0)[:-1] @ v[lo:n, h // 4].double(), dtype, (window, b, h))


# ---- latent attention ---------------------------------------------------------------------------------------------------
LATENT = [  # T, H, dim, rot, vdim, rank, block
    (70, 3, 24, 8, 40, 72, 16), (130, 2, 64, 32, 64, 64, 32), (90, 18, 128, 64, 96, 264, 64), (75, 5, 22, 6, 26, 50, 16),
    (140, 2, 32, 40, 160, 128, 16), (65, 4, 40, 24, 48, 200, 32), (60, 2, 16, 8, 16, 512, 16), (50, 1, 200, 56, 256, 96, 16),
    (40, 2, 16, 80, 24, 40, 16), (200, 16, 32, 16, 32, 120, 64)]


def latent_case(T, H, dim, rot, vdim, rank, dtype, seed=0, needle=None):
    """Projection rows and weights; needle = (query, key): the pair's unrotated parts point at each other."""
    eps, base = 1e-4, 300.0
    proj = rand(T, H * (dim + rot) + rank + rot, seed=seed + 1, dtype=dtype)
    norm = (1 + 0.2 * rand(rank, seed=seed + 2)).to(dtype)
    uk, uv = (rand(H * n, rank, seed=seed + 3 + i, dtype=dtype, scale=rank ** -0.5) for i, n in enumerate((dim, vdim)))
    if needle:
        i, j = needle
        proj *= 0.05
        proj[j, H * (dim + rot):H * (dim + rot) + rank] = 0
        proj[j, H * (dim + rot)] = 1.0                 # normalised, the latent is sqrt(rank) in its first element
        norm = torch.ones(rank, dtype=dtype)
        uk[:, 0] = 1.0
        proj[i, :H * (dim + rot)] = 12.0 / (dim ** 0.5)
        proj[i, :H * (dim + rot)].view(H, dim + rot)[:, dim:] = 0
    freqs, mag = o.rotary_frequencies(rot, base)
    d = proj.double()
    latent = o.rms(d[:, H * (dim + rot):H * (dim + rot) + rank], norm.double(), eps)
    keys, queries, krot = [], [], []
    for t in range(T):
        r = o.rotate_interleaved(d[t:t + 1, -rot:], t, freqs, mag, rot)
        q = d[t, :H * (dim + rot)].view(H, dim + rot)
        krot.append(r[0])
        keys.append(torch.cat([(uk.double() @ latent[t]).view(H, dim), r.expand(H, rot)], 1))
        queries.append(torch.cat([q[:, :dim], o.rotate_interleaved(q[:, dim:], t, freqs, mag, rot)], 1))
    values = (latent @ uv.double().T).view(T, H, vdim)
    return proj, norm, uk, uv, latent, torch.stack(krot), torch.stack(queries), torch.stack(keys), values, eps, base


class LatentRun:
    """One sequence in a scattered latent cache; rows that nobody wrote hold garbage in front of the padding."""

    def __init__(self, case, H, dim, rot, vdim, rank, bs, dtype):
        proj, self.norm, uk, uv, *_, self.eps, base = case
        T = proj.shape[0]
        self.H, self.dim, self.rot, self.vdim, self.rank, self.bs, self.dtype = H, dim, rot, vdim, rank, bs, dtype
        self.proj, self.norm = proj.cuda(), self.norm.cuda()
        self.expand = torch.cat([uk, uv]).cuda()
        self.into = uk.view(H, dim, rank).transpose(1, 2).contiguous().cuda()
        self.out_of = uv.view(H, vdim, rank).contiguous().cuda()
        self.rot_at, self.row = ops.latent_row(rank, rot, dtype)
        nb = -(-T // bs)
        self.table = torch.randperm(nb + 3, generator=torch.Generator().manual_seed(9))[:nb].to(torch.int32).cuda()
        self.cache = torch.full((nb + 3, 1, bs, self.row), 1e3, dtype=dtype, device=DEV)
        self.cache[..., rank:self.rot_at], self.cache[..., self.rot_at + rot:] = 0, 0
        self.cos_sin = rotary_table(RotarySpec(rot, base), T).cuda()

    def store(self, at, n, q_row, rot_q, plain, active=True):
        pos = torch.arange(at, at + n, device=DEV)
        slots = self.table[pos // self.bs].long() * self.bs + pos % self.bs if active else torch.full_like(pos, -1)
        return ops.latent_store(self.proj[at:at + n].contiguous(), self.norm, self.cos_sin, pos, slots, self.cache, self.H,
                                self.dim, self.rot_at, self.eps, q_row, rot_q, plain)

    def absorbed_query(self, at, n):
        q = self.store(at, n, self.row, self.rot_at, False)
        x = self.proj[at:at + n, :self.H * (self.dim + self.rot)].view(n, self.H, -1)
        return ops.head_linear(x, self.into, q)

    def read_out(self, o_latent):
        n = o_latent.shape[0]
        y = torch.empty(n, self.H, self.vdim, dtype=self.dtype, device=DEV)
        return ops.head_linear(o_latent, self.out_of, y).view(n, -1)

    def portion(self, at, n, scale, form):
        layout = span(at, n, self.table, self.bs)
        if form == "expanded":
            width = ops.latent_prefill_query_row(self.dim, self.rot, self.vdim, self.rank, self.dtype)
            q = self.store(at, n, width, self.dim, True)
            rows = ops.latent_gather(self.cache, layout, self.rank, self.rot, self.rot_at)
            kv = (rows[:, :self.rank].float() @ self.expand.float().T).to(self.dtype)
            return ops.latent_attention_prefill(q, kv, rows[:, self.rank:], layout, self.dim, self.vdim, scale)
        q = self.absorbed_query(at, n)
        if form == "row by row":
            return self.read_out(ops.latent_attention_decode(q, self.cache, *layout.row_tables(), self.rank, self.rot_at, scale))
        out = ops.attention_prefill(q, self.cache, self.cache, layout, self.row, self.rank, scale)
        return self.read_out(out.view(n, self.H, self.rank))


def latent_forms(run):
    wide = ops.latent_prefill_query_row(run.dim, run.rot, run.vdim, run.rank, run.dtype)
    return ["absorbed", "row by row"] + (["expanded"] if wide else [])


def test_every_latent_form_is_among_the_cases():
    wide = [bool(ops.latent_prefill_query_row(d, r, v, k, torch.bfloat16)) for _, _, d, r, v, k, _ in LATENT]
    rows = [ops.latent_row(k, r, torch.bfloat16) for _, _, _, r, _, k, _ in LATENT]
    assert True in wide and False in wide and {a for a, _ in rows} >= {64, 128, 256, 512}
    assert {b - a for a, b in rows} >= {32, 64, 80}
    assert not ops.latent_prefill_query_row(64, 32, 64, 64, torch.float32)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,H,dim,rot,vdim,rank,bs", LATENT)
def test_latent_attention(dtype, T, H, dim, rot, vdim, rank, bs):
    case = latent_case(T, H, dim, rot, vdim, rank, dtype)
    *_, latent, krot, queries, keys, values, _, _ = case
    scale = 1.5 * (dim + rot) ** -0.5
    want = o.attend(queries, keys, values, scale).reshape(T, H * vdim)
    run = LatentRun(case, H, dim, rot, vdim, rank, bs, dtype)
    for form in latent_forms(run):
        print(f"latent {form} T={T} H={H} dim={dim} rot={rot} vdim={vdim} rank={rank} {dtype}", flush=True)
        close(run.portion(0, T, scale, form), want, dtype, form)
        at = 0
        for n in (2, 3, 17, 16, 1, 31, T):
            n = min(n, T - at)
            if n:
                close(run.portion(at, n, scale, form), want[at:at + n], dtype, f"{form} {at}+{n}")
            at += n
    pos = torch.arange(T, device=DEV)
    got = run.cache.view(-1, run.row)[run.table[pos // bs].long() * bs + pos % bs]
    close(got[:, :rank], latent, dtype, "latent rows")
    close(got[:, run.rot_at:run.rot_at + rot], krot, dtype, "rotated rows")
    assert torch.count_nonzero(got[:, rank:run.rot_at]) == 0 and torch.count_nonzero(got[:, run.rot_at + rot:]) == 0
    before = run.cache.clone()
    q = run.store(T - 1, 1, run.row, run.rot_at, False, active=False)          # an idle row writes nothing
    assert torch.equal(run.cache, before)
    close(q[0, :, run.rot_at:run.rot_at + rot], queries[T - 1, :, dim:], dtype, "rotated queries")


@pytest.mark.parametrize("dtype", DTYPES)
def test_latent_key_far_away_stands_out(dtype):
    T, H, dim, rot, vdim, rank, bs = 330, 2, 32, 16, 32, 64, 16
    for i, j in ((329, 0), (329, 16), (329, 15), (300, 300), (300, 299), (300, 288), (300, 287), (64, 63), (63, 0)):
        case = latent_case(T, H, dim, rot, vdim, rank, dtype, needle=(i, j))
        values = case[8]
        run = LatentRun(case, H, dim, rot, vdim, rank, bs, dtype)
        run.portion(0, T, 0.3, "absorbed")             # fills the cache
        for form in latent_forms(run):
            print(f"latent needle {i} {j} {form} {dtype}", flush=True)
            for at in (i, max(0, i - 37)):
                got = run.portion(at, i - at + 1, 0.3, form)[-1]
                assert (got.double().cpu() - values[j].reshape(-1)).abs().max() < 3e-2, (i, j, form, at)
            if j < i:                                  # the query in front of it does not point there
                got = run.portion(i - 1, 1, 0.3, form)[-1]
                assert (got.double().cpu() - values[j].reshape(-1)).abs().max() > 0.1


def test_latent_decode_over_context_splits_and_head_tiles():
    dtype, bs = torch.bfloat16, 64
    for rank, rot, H, T in ((512, 64, 20, 2600), (64, 32, 3, 2600), (128, 64, 16, 1100), (256, 32, 33, 1100)):
        print(f"latent long decode rank={rank} rot={rot} H={H}", flush=True)
        rot_at, row = ops.latent_row(rank, rot, dtype)
        nb = -(-T // bs)
        table = torch.randperm(nb + 2, generator=torch.Generator().manual_seed(1))[:nb].to(torch.int32)
        cache = rand(nb + 2, 1, bs, row, seed=2, dtype=dtype)
        cache[..., rank:rot_at], cache[..., rot_at + rot:] = 0, 0
        ctx = torch.tensor([T, 1, 63, 65, T - 1, 513], dtype=torch.int32)
        q = rand(len(ctx), H, row, seed=3, dtype=dtype, scale=0.5)
        got = ops.latent_attention_decode(q.cuda(), cache.cuda(), table.cuda().repeat(len(ctx), 1).contiguous(), ctx.cuda(), rank,
                                          rot_at, 0.1)
        rows = cache[table.long()].reshape(-1, row).double()
        for b, n in enumerate(ctx.tolist()):
            p = torch.softmax(q[b].double() @ rows[:n].T * 0.1, -1)
            close(got[b], p @ rows[:n, :rank], dtype, (rank, b))


def test_latent_ragged_pass_equals_each_segment_alone():
    H, dim, rot, vdim, rank, bs, dtype = 4, 40, 24, 48, 120, 16, torch.bfloat16
    portions = [(0, 300), (37, 150), (0, 1), (250, 2), (128, 128)]
    total = [s + n for s, n in portions]
    nb = [-(-t // bs) for t in total]
    order = torch.randperm(sum(nb), generator=torch.Generator().manual_seed(2)).tolist()
    rot_at, row = ops.latent_row(rank, rot, dtype)
    cache = rand(sum(nb), 1, bs, row, seed=7, dtype=dtype).cuda()
    cache[..., rank:rot_at], cache[..., rot_at + rot:] = 0, 0
    segs = [(s, n, [order.pop() for _ in range(m)], i) for i, ((s, n), m) in enumerate(zip(portions, nb))]
    width = ops.latent_prefill_query_row(dim, rot, vdim, rank, dtype)
    q = rand(sum(n for _, n in portions), H, width, seed=3, dtype=dtype)
    q[..., dim + rot:] = 0
    q, w = q.cuda(), rand(H * (dim + vdim), rank, seed=4, dtype=dtype, scale=rank ** -0.5).cuda()

    def attend(qs, layout):
        rows = ops.latent_gather(cache, layout, rank, rot, rot_at)
        return ops.latent_attention_prefill(qs, torch.nn.functional.linear(rows[:, :rank], w), rows[:, rank:], layout, dim, vdim, 0.1)
    print("latent ragged", flush=True)
    got, at = attend(q, ops.PromptPass(segs, bs, torch.device(DEV))), 0
    for seg in segs:
        alone = attend(q[at:at + seg[1]].contiguous(), ops.PromptPass([seg], bs, torch.device(DEV)))
        close(got[at:at + seg[1]], alone.double().cpu(), dtype, seg[:2])
        at += seg[1]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows,H,n_in,n_out", [(1, 4, 128, 512), (20, 3, 40, 24), (37, 2, 512, 128), (5, 2, 21, 7), (16, 1, 300, 50)])
def test_head_linear(dtype, rows, H, n_in, n_out):
    print(f"head_linear {rows} {H} {n_in} -> {n_out} {dtype}", flush=True)
    x, w = rand(rows, H * (n_in + 8) + 16, seed=1, dtype=dtype), rand(H, n_out, n_in, seed=2, dtype=dtype, scale=n_in ** -0.5)
    y = torch.full((rows, H, n_out + 5), 7.0, dtype=dtype, device=DEV)
    xv = x.cuda()[:, :H * (n_in + 8)].view(rows, H, n_in + 8)
    ops.head_linear(xv, w.cuda(), y)
    want = torch.stack([x[:, h * (n_in + 8):h * (n_in + 8) + n_in].double() @ w[h].double().T for h in range(H)], 1)
    close(y[..., :n_out], want, dtype)
    assert (y[..., n_out:] == 7.0).all()


# ---- selective scan -------------------------------------------------------------------------------------------------------
SCANS = [  # T, channels, states, rank, taps
    (1, 40, 16, 8, 4), (37, 88, 24, 8, 4), (150, 300, 16, 24, 3), (100, 50, 5, 3, 2), (45, 64, 130, 16, 1), (130, 20, 256, 8, 16),
    (700, 72, 64, 16, 4), (90, 33, 33, 5, 7), (64, 520, 1, 40, 4)]


def scan_case(T, C, N, rank, taps, dtype, seed=0):
    xz, sel = rand(T, 2 * C, seed=seed + 1, dtype=dtype), rand(T, rank + 2 * N, seed=seed + 2, dtype=dtype)
    conv, bias = rand(C, taps, seed=seed + 3, dtype=dtype, scale=taps ** -0.5), rand(C, seed=seed + 4, dtype=dtype, scale=0.3)
    up, dt_b = rand(C, rank, seed=seed + 5, dtype=dtype, scale=rank ** -0.5), (rand(C, seed=seed + 6) * 1.5 - 2.5).to(dtype)
    a_log = (torch.arange(1.0, N + 1).log() - 2.5 + rand(C, N, seed=seed + 7)).to(dtype)
    return xz, sel, conv, bias, up, dt_b, a_log, (1 + 0.5 * rand(C, seed=seed + 8)).to(dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,C,N,rank,taps", SCANS)
def test_selective_scan_prefill_portions_and_decode(dtype, T, C, N, rank, taps):
    print(f"scan T={T} C={C} N={N} rank={rank} taps={taps} {dtype}", flush=True)
    case = scan_case(T, C, N, rank, taps, dtype)
    xz, sel, conv, bias, up, dt_b, a_log, skip = case
    d = [t.double() for t in case]
    x = o.silu(o.short_conv(d[0][:, :C], d[2], d[3]))
    xr = x.to(dtype).double()                              # the scan is given the convolution's result as it is stored
    dt = o.softplus(d[1][:, :rank] @ d[4].T + d[5])
    y, S = o.selective_scan(xr, dt, -torch.exp(d[6]), d[1][:, rank:rank + N], d[1][:, rank + N:], d[7])
    want = y * o.silu(d[0][:, C:])
    padded = torch.cat([torch.zeros(max(0, taps - 1 - T), C).double(), d[0][:, :C]])
    tail_want = padded[len(padded) - (taps - 1):]
    xz, sel, conv, bias, up, dt_b, a_log, skip = (t.cuda() for t in case)
    got_dt = ops.scan_dt(sel[:, :rank], up, dt_b)
    close(got_dt, dt, torch.float32, "dt")
    slots = 3
    for piece in {ops.scan_piece_rows(T, C, N), 32}:
        for cuts in ([T], [2] * (T // 2) + [T % 2], [T // 3, 16, T]):
            state, tail = torch.full((slots, N, C), 1e3, device=DEV), torch.full((slots, taps - 1, C), 1e3, device=DEV)
            xs, out = torch.empty(T, C, dtype=dtype, device=DEV), torch.empty(T, C, dtype=dtype, device=DEV)
            at = 0
            for n in cuts:
                n = min(n, T - at)
                if n > 0:
                    s = slice(at, at + n)
                    one = ops.PromptPass([(at, n, range(T), 1)], 1, torch.device(DEV))
                    xs[s] = ops.conv_silu(xz[s, :C], conv, bias, tail, one, piece)
                    given = xr[s].to(dtype).cuda().contiguous()
                    out[s] = ops.scan_prefill(given, got_dt[s], sel[s, rank:], xz[s, C:], a_log, skip, xz[s, :C], state, tail, one,
                                              piece)
                    at += n
            assert at == T
            close(xs, x, dtype, f"conv {cuts[:2]}")
            close(out, want, dtype, f"out {cuts[:2]} piece {piece}")
            close(state[1], S.T, torch.float32, "state")
            assert torch.equal(tail[1].cpu().double(), tail_want)
            assert (state[0] == 1e3).all() and (state[2] == 1e3).all() and (tail[0] == 1e3).all() and (tail[2] == 1e3).all()
    # token by token, an idle row and foreign slots beside it
    state, tail = torch.full((slots, N, C), 1e3, device=DEV), torch.full((slots, taps - 1, C), 1e3, device=DEV)
    active, slot = torch.tensor([True, False], device=DEV), torch.tensor([2, 0], dtype=torch.int32, device=DEV)
    steps = min(T, 40)
    for t in range(steps):
        pos, two = torch.tensor([t, t], device=DEV), lambda a: a[t:t + 1].repeat(2, 1)
        xs = ops.conv_step(two(xz)[:, :C], conv, bias, tail, slot, pos, active)
        given = two(xr.to(dtype).cuda())
        out = ops.scan_step(given, two(got_dt), two(sel)[:, rank:], two(xz)[:, C:], a_log, skip, state, slot, pos, active)
        close(xs[0], x[t], dtype, f"conv step {t}")
        close(out[0], want[t], dtype, f"step {t}")
        assert torch.count_nonzero(out[1]) == 0 and torch.count_nonzero(xs[1]) == 0
    assert (state[:2] == 1e3).all() and (tail[:2] == 1e3).all()
    if steps == T:
        close(state[2], S.T, torch.float32, "state after steps")
        assert torch.equal(tail[2].cpu().double(), tail_want)


@pytest.mark.parametrize("rows,channels,rank", [(512, 128, 64), (700, 200, 72), (1030, 36, 8), (513, 300, 128), (600, 30, 24)])
def test_scan_step_sizes_of_long_passes(rows, channels, rank):
    print(f"scan_dt {rows}x{channels} rank {rank}", flush=True)
    low, up = rand(rows, rank + 16, seed=1, dtype=torch.bfloat16), rand(channels, rank, seed=2, dtype=torch.bfloat16)
    b = rand(channels, seed=3, dtype=torch.bfloat16)
    got = ops.scan_dt(low.cuda()[:, :rank], up.cuda(), b.cuda())
    close(got, o.softplus(low[:, :rank].double() @ up.double().T + b.double()), torch.float32)


@pytest.mark.parametrize("dtype", DTYPES)
def test_one_state_entry_lives_on(dtype):
    """A single token writes the state and slow decays keep it: the read-out far behind it, over pieces, portions and steps,
    is what it wrote; a convolution tap that reaches over a portion's start shows."""
    T, C, N = 400, 24, 20
    for j in (0, 1, 31, 32, 63, 64, 127):
        print(f"scan needle {j} {dtype}", flush=True)
        x, dt = torch.zeros(T, C), torch.full((T, C), 1e-4)
        x[j], dt[j] = 3.0, 1.0
        bc = torch.zeros(T, 2 * N)
        bc[j, 7], bc[T - 1, N + 7] = 2.0, 1.5                     # written and read in one entry
        a_log, z = torch.full((C, N), -4.0), torch.full((T, C), 1.0)
        want = 3.0 * 2.0 * 1.5 * torch.exp(-torch.exp(torch.tensor(-4.0)) * 1e-4 * (T - 1 - j)) * o.silu(torch.tensor(1.0))
        x, bc, z, a_log = (t.to(dtype).cuda() for t in (x, bc, z, a_log))
        dt, skip = dt.cuda(), torch.zeros(C, dtype=dtype, device=DEV)
        for cuts in ([T], [j + 1, T - j - 1], [100, 2, T - 102], [T - 2, 2]):
            state, tail, at = torch.full((1, N, C), 9.0, device=DEV), torch.full((1, 3, C), 9.0, device=DEV), 0
            for n in cuts:
                s = slice(at, at + n)
                one = ops.PromptPass([(at, n, range(T), 0)], 1, torch.device(DEV))
                out = ops.scan_prefill(x[s], dt[s], bc[s], z[s], a_log, skip, x[s], state, tail, one, 32)
                at += n
            assert (out[-1].float().cpu() - want).abs().max() < 2e-2 * want, (j, cuts)


@pytest.mark.parametrize("dtype", DTYPES)
def test_scan_steps_of_a_wide_batch_equal_each_row_alone(dtype):
    """More rows than one workgroup takes, some idle, fresh and running ones, slots in any order."""
    B, C, N, rank, taps = 37, 100, 20, 8, 4
    print(f"scan wide step {dtype}", flush=True)
    xz, sel, conv, bias, up, dt_b, a_log, skip = (t.cuda() for t in scan_case(B, C, N, rank, taps, dtype))
    s0, t0 = rand(B + 3, N, C, seed=5).cuda(), rand(B + 3, taps - 1, C, seed=6).cuda()
    slot = torch.randperm(B + 3, generator=torch.Generator().manual_seed(3))[:B].to(torch.int32).cuda()
    pos, active = torch.arange(B, device=DEV) % 5, torch.arange(B, device=DEV) % 7 != 3
    dt = ops.scan_dt(sel[:, :rank], up, dt_b)

    def go(rows, state, tail):
        x = ops.conv_step(xz[rows, :C], conv, bias, tail, slot[rows], pos[rows], active[rows])
        return ops.scan_step(x, dt[rows], sel[rows, rank:], xz[rows, C:], a_log, skip, state, slot[rows], pos[rows], active[rows])
    sa, ta, sb, tb = s0.clone(), t0.clone(), s0.clone(), t0.clone()
    got = go(slice(0, B), sa, ta)
    want = torch.cat([go(slice(i, i + 1), sb, tb) for i in range(B)])
    assert torch.equal(got, want) and torch.equal(sa, sb) and torch.equal(ta, tb)
    idle = slot[~active].long()
    assert torch.equal(sa[idle], s0[idle]) and torch.count_nonzero(got[~active]) == 0 and not torch.equal(sa, s0)


def test_scan_ragged_pass_equals_each_sequence_alone():
    C, N, rank, taps, dtype = 80, 20, 8, 4, torch.bfloat16
    portions = [(0, 300), (37, 150), (0, 1), (250, 2), (128, 128), (5, 1)]
    T = sum(n for _, n in portions)
    xz, sel, conv, bias, up, dt_b, a_log, skip = (t.cuda() for t in scan_case(T, C, N, rank, taps, dtype))
    segs = [(s, n, range(s + n), i) for i, (s, n) in enumerate(portions)]
    s0, t0 = rand(len(segs), N, C, seed=5).cuda(), rand(len(segs), taps - 1, C, seed=6).cuda()
    dt = ops.scan_dt(sel[:, :rank], up, dt_b)

    def go(rows, layout, state, tail, piece=32):
        x = ops.conv_silu(xz[rows, :C], conv, bias, tail, layout, piece)
        return ops.scan_prefill(x, dt[rows], sel[rows, rank:], xz[rows, C:], a_log, skip, xz[rows, :C], state, tail, layout, piece)
    print("scan ragged", flush=True)
    state, tail = s0.clone(), t0.clone()
    layout = ops.PromptPass(segs, 1, torch.device(DEV))
    assert layout.pieces(32)[2]
    out, at = go(slice(0, T), layout, state, tail), 0
    for i, seg in enumerate(segs):
        sa, ta = s0.clone(), t0.clone()
        alone = go(slice(at, at + seg[1]), ops.PromptPass([seg], 1, torch.device(DEV)), sa, ta, 512)     # in one piece
        close(out[at:at + seg[1]], alone.double().cpu(), dtype, i)
        close(state[i], sa[i].double().cpu(), torch.float32, i)
        assert torch.equal(tail[i], ta[i])
        at += seg[1]


def test_argument_checks_of_these_kernels():
    f = lambda *s: torch.zeros(*s, device=DEV)
    with pytest.raises(_lib.AwqHipError, match="streams"):
        ops.hyper_norm(f(1, 9, 8), 1e-5, next_weight=f(8))
    with pytest.raises(_lib.AwqHipError, match="states"):
        ops.scan_step(f(1, 8), f(1, 8), f(1, 600), f(1, 8), f(8, 300), f(8), f(1, 300, 8),
                      torch.zeros(1, dtype=torch.int32, device=DEV), torch.zeros(1, dtype=torch.long, device=DEV),
                      torch.ones(1, dtype=torch.bool, device=DEV))
    with pytest.raises(_lib.AwqHipError, match="taps"):
        ops.conv_step(f(1, 8), f(8, 20), f(8), f(1, 19, 8), torch.zeros(1, dtype=torch.int32, device=DEV),
                      torch.zeros(1, dtype=torch.long, device=DEV), torch.ones(1, dtype=torch.bool, device=DEV))
    with pytest.raises(_lib.AwqHipError):
        ops.latent_attention_decode(f(1, 2, 1200), f(1, 1, 16, 1200), torch.zeros(1, 1, dtype=torch.int32, device=DEV),
                                    torch.ones(1, dtype=torch.int32, device=DEV), 1100, 1100, 1.0)
