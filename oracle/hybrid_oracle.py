"""Plain, slow restatement of the mechanisms of config-described hybrid decoders, on CPU tensors.

TEST INFRASTRUCTURE, NOT PRODUCT.  One function per mechanism, written from the equations with explicit loops over
tokens and keys; float64 by default.  `gafulix_logits` and `roletar_logits` compose them for a checkpoint given as
(config dictionary, {tensor name: tensor}).  Nothing here is imported by the product and nothing of the product is imported here."""
from __future__ import annotations

import math

import torch


def rms(x, weight=None, eps=0.0):
    y = x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)
    return y if weight is None else y * weight


def silu(x):
    return x / (1.0 + torch.exp(-x))


# ---- rotary -----------------------------------------------------------------------------------------------------
def rotary_frequencies(dims, base, scaling=None):
    """(angular frequency of every pair, factor on cos and sin); `scaling` is the YaRN dictionary or None."""
    freqs = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    if not scaling:
        return freqs, 1.0

    def pair_of(turns):        # the (fractional) pair index that makes `turns` rotations over the original length
        return dims * math.log(scaling["original"] / (2.0 * math.pi * turns)) / (2.0 * math.log(base))
    lo = max(math.floor(pair_of(scaling["fast"])), 0)
    hi = min(math.ceil(pair_of(scaling["slow"])), dims - 1)
    out = []
    for i, f in enumerate(freqs):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(f / scaling["factor"] * ramp + f * (1.0 - ramp))
    return out, 0.1 * math.log(scaling["factor"]) + 1.0


def rotate_interleaved(x, position, freqs, magnitude, dims):
    """x [heads, dim] at one position: pairs (2i, 2i + 1) of the first `dims` dimensions are rotated."""
    y = x.clone()
    for i, f in enumerate(freqs):
        a = position * f
        c, s = math.cos(a) * magnitude, math.sin(a) * magnitude
        u, v = x[:, 2 * i], x[:, 2 * i + 1]
        y[:, 2 * i] = u * c - v * s
        y[:, 2 * i + 1] = v * c + u * s
    assert 2 * len(freqs) == dims
    return y


# ---- attention --------------------------------------------------------------------------------------------------
def visible(i, j, chunk=None, window=None):
    """Whether the token at position i sees the key at position j."""
    return j <= i and (not chunk or i // chunk == j // chunk) and (not window or i - j < window)


def attend(q, k, v, scale, chunk=None, window=None, sink=None):
    """q [T, H, dim], k [T, G, dim], v [T, G, vdim] of one sequence from position 0; returns [T, H, vdim].
    sink [H]: a further, unscaled score per head whose share of the softmax goes nowhere."""
    T, H, _ = q.shape
    G = k.shape[1]
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    for i in range(T):
        js = [j for j in range(T) if visible(i, j, chunk, window)]
        for h in range(H):
            g = h // (H // G)
            s = (k[js, g] @ q[i, h]) * scale
            top = s.max() if sink is None else torch.maximum(s.max(), sink[h])
            p = torch.exp(s - top)
            total = p.sum() if sink is None else p.sum() + torch.exp(sink[h] - top)
            out[i, h] = (p / total) @ v[js, g]
    return out


def attention_mixer(h, w, cfg, eps):
    T = h.shape[0]
    H, G, dim, vdim = cfg["heads"], cfg["kv_heads"], cfg["dim"], cfg["vdim"]
    q = rms(h @ w["q"].T + w["q.b"], w["q.norm"], eps).view(T, H, dim)
    k = rms(h @ w["k"].T + w["k.b"], w["k.norm"], eps).view(T, G, dim)
    v = (h @ w["v"].T + w["v.b"]).view(T, G, vdim)
    rot = cfg.get("rot")
    if rot:
        freqs, mag = rotary_frequencies(rot["dims"], rot["base"], rot.get("scaling"))
        q = torch.stack([rotate_interleaved(q[t], t, freqs, mag, rot["dims"]) for t in range(T)])
        k = torch.stack([rotate_interleaved(k[t], t, freqs, mag, rot["dims"]) for t in range(T)])
    chunk = (cfg.get("mask") or {}).get("size")
    return attend(q, k, v, cfg["scale"], chunk).reshape(T, H * vdim) @ w["o"].T


def sink_attention_mixer(h, w, cfg, eps):
    """Grouped heads without rotation, a sliding window, a sink per head."""
    T = h.shape[0]
    H, G, dim, vdim = cfg["heads"], cfg["kv_heads"], cfg["dim"], cfg["vdim"]
    q, k, v = (h @ w["q"].T).view(T, H, dim), (h @ w["k"].T).view(T, G, dim), (h @ w["v"].T).view(T, G, vdim)
    window = (cfg.get("mask") or {}).get("size")
    return attend(q, k, v, cfg["scale"], window=window, sink=w["sink"]).reshape(T, H * vdim) @ w["o"].T


def latent_attention_mixer(h, w, cfg, eps):
    """Keys and values of all heads from one normalised latent per token, plus one rotated key part that the heads share."""
    T = h.shape[0]
    H, dim, rd, vdim, rank = cfg["heads"], cfg["dim"], cfg["rot_dim"], cfg["vdim"], cfg["kv_rank"]
    freqs, mag = rotary_frequencies(rd, cfg["rot"]["base"])
    q = (h @ w["q"].T).view(T, H, dim + rd)
    down = h @ w["dkv"].T
    latent = rms(down[:, :rank], w["dkv.norm"], eps)
    k_nope, v = (latent @ w["uk"].T).view(T, H, dim), (latent @ w["uv"].T).view(T, H, vdim)
    keys, queries = [], []
    for t in range(T):
        k_rot = rotate_interleaved(down[t:t + 1, rank:], t, freqs, mag, rd)
        keys.append(torch.cat([k_nope[t], k_rot.expand(H, rd)], dim=1))
        queries.append(torch.cat([q[t, :, :dim], rotate_interleaved(q[t, :, dim:], t, freqs, mag, rd)], dim=1))
    return attend(torch.stack(queries), torch.stack(keys), v, cfg["scale"]).reshape(T, H * vdim) @ w["o"].T


# ---- selective scan (Gu and Dao, "Mamba: Linear-Time Sequence Modeling with Selective State Spaces") -------------------
def short_conv(x, weight, bias, before=None):
    """x [T, C], weight [C, taps] (last column: the current token), `before` [taps - 1, C]: the inputs ahead of x (zeros)."""
    T, C = x.shape
    taps = weight.shape[1]
    padded = torch.cat([torch.zeros(taps - 1, C, dtype=x.dtype) if before is None else before, x])
    out = bias.expand(T, C).clone()
    for k in range(taps):
        out = out + weight[:, k] * padded[k:k + T]
    return out


def softplus(z):
    return torch.clamp(z, min=0.0) + torch.log1p(torch.exp(-z.abs()))


def selective_scan(x, dt, A, B, C, D, state=None):
    """x, dt [T, channels], A [channels, N] (negative), B, C [T, N], D [channels]; state [channels, N] (zero if not given).
    Returns (y [T, channels], the state after the last token)."""
    S = torch.zeros_like(A) if state is None else state.clone()
    out = torch.zeros_like(x)
    for t in range(x.shape[0]):
        S = torch.exp(dt[t, :, None] * A) * S + (dt[t] * x[t])[:, None] * B[t]
        out[t] = S @ C[t] + D * x[t]
    return out, S


def mamba1_mixer(h, w, cfg, eps):
    inner, rank, n = cfg["inner"], cfg["dt_rank"], cfg["state"]
    x, z = (h @ w["in"].T).split([inner, inner], dim=1)
    x = silu(short_conv(x, w["conv"], w["conv.b"]))
    low, B, C = (x @ w["x"].T).split([rank, n, n], dim=1)
    dt = softplus(low @ w["dt"].T + w["dt.b"])
    y, _ = selective_scan(x, dt, -torch.exp(w["A_log"]), B, C, w["D"])
    return (y * silu(z)) @ w["o"].T


# ---- gated linear attention -------------------------------------------------------------------------------------
def channel_decay(z, tau):
    return (1.0 / (1.0 + torch.exp(-z))) ** (1.0 / tau)


def gla_scan(q, k, v, decay, state=None):
    """q, k, decay [T, H, dim], v [T, H, vdim]; state [H, dim, vdim] (zero if not given).  Returns (o [T, H, vdim], the
    state after the last token): the state decays per key channel, takes the outer product k v, and is read by q."""
    T, H, dim = q.shape
    S = torch.zeros(H, dim, v.shape[2], dtype=q.dtype) if state is None else state.clone()
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    for t in range(T):
        S = decay[t].unsqueeze(-1) * S + k[t].unsqueeze(-1) * v[t].unsqueeze(-2)
        out[t] = (S * q[t].unsqueeze(-1)).sum(dim=1)
    return out, S


def gla_mixer(h, w, cfg, eps):
    T = h.shape[0]
    H, dim, vdim = cfg["heads"], cfg["dim"], cfg["vdim"]
    q = (h @ w["q"].T).view(T, H, dim) * dim ** -0.5
    k = (h @ w["k"].T).view(T, H, dim)
    v = (h @ w["v"].T).view(T, H, vdim)
    z = ((h @ w["a1"].T) @ w["a2"].T + w["a2.b"]).view(T, H, dim)
    o, _ = gla_scan(q, k, v, channel_decay(z, cfg["tau"]))
    o = rms(o, w["norm"], eps).reshape(T, H * vdim) * silu(h @ w["g"].T)
    return o @ w["o"].T


# ---- mixture of experts -----------------------------------------------------------------------------------------
def route(h, router, top):
    """Per token the `top` experts with the largest sigmoid scores, and those scores as they are."""
    s = 1.0 / (1.0 + torch.exp(-(h @ router.T)))
    picks = []
    for t in range(h.shape[0]):
        order = sorted(range(s.shape[1]), key=lambda e: (-s[t, e].item(), e))[:top]
        picks.append([(e, s[t, e]) for e in order])
    return picks


def moe(h, w, cfg):
    """The score multiplies what goes INTO the expert; expert outputs are summed as they are."""
    out = torch.zeros_like(h)
    for t, picks in enumerate(route(h, w["router"], cfg["router"]["top"])):
        for e, s in picks:
            u = h[t] * s
            out[t] += w[f"e{e}.down"] @ (silu(w[f"e{e}.gate"] @ u) * (w[f"e{e}.up"] @ u))
    return out


def relu2_mlp(h, w):
    return torch.clamp(h @ w["up"].T, min=0.0) ** 2 @ w["down"].T


# ---- hyper-connections -------------------------------------------------------------------------------------------
def hyper_read(xs, w_in):
    """The input of a sublayer from the streams xs [S, T, width]."""
    return sum(w_in[s] * xs[s] for s in range(len(xs)))


def hyper_write(xs, mix, w_out, y):
    """Every stream anew from all the old ones (mix[from, to]) and the sublayer's output."""
    n = len(xs)
    return torch.stack([sum(mix[s, t] * xs[s] for s in range(n)) + w_out[t] * y for t in range(n)])


def softcap(logits, cap):
    return cap * torch.tanh(logits / cap)


# ---- the model --------------------------------------------------------------------------------------------------
def layer_schedule(config):
    """[(layer index, whether the embedding output is added in front of it)] in execution order."""
    n = len(config["layers"])
    loop = config.get("loop")
    if not loop:
        return [(i, False) for i in range(n)]
    a, b, times = loop["start"], loop["stop"], loop["times"]
    runs = [(i, False) for i in range(a)]
    for rep in range(times):
        runs += [(i, rep > 0 and i == a) for i in range(a, b)]
    return runs + [(i, False) for i in range(b, n)]


def _sub(weights, prefix, dtype):
    return {k[len(prefix):]: t.to(dtype) for k, t in weights.items() if k.startswith(prefix)}


def gafulix_logits(config, weights, tokens, dtype=torch.float64, trace=None):
    """tokens: list of ids of one sequence.  Returns logits [T, vocab]; `trace` (a list) receives the residual stream
    after every layer run."""
    eps = config["norm"]["eps"]
    w = lambda name: weights[name].to(dtype)
    emb = w("embed")[torch.tensor(tokens)]
    x = emb.clone()
    for i, add in layer_schedule(config):
        layer = config["layers"][i]
        if add:
            x = x + emb
        mix = _sub(weights, f"l{i}.mix.", dtype)
        mixer = {"attention": attention_mixer, "gla": gla_mixer}[layer["type"]]
        x = x + rms(mixer(rms(x, w(f"l{i}.norm1"), eps), mix, layer["mixer"], eps), w(f"l{i}.norm1b"), eps)
        if layer.get("mlp"):
            y = moe(rms(x, w(f"l{i}.norm2"), eps), _sub(weights, f"l{i}.mlp.", dtype), layer["mlp"])
            x = x + rms(y, w(f"l{i}.norm2b"), eps)
        if trace is not None:
            trace.append(x.clone())
    return rms(x, w("final.norm"), eps) @ w("head").T


def roletar_logits(config, weights, tokens, dtype=torch.float64, trace=None):
    """As gafulix_logits.  `trace` receives the sum of the streams."""
    eps = config["norm"]["eps"]
    w = lambda name: weights[name].to(dtype)
    emb = w("embed")[torch.tensor(tokens)]
    xs = torch.stack([emb] * config["streams"])
    for i, _ in layer_schedule(config):
        layer = config["layers"][i]
        mix = _sub(weights, f"l{i}.mix.", dtype)
        mixer = {"attention": sink_attention_mixer, "latent_attention": latent_attention_mixer,
                 "mamba1": mamba1_mixer}[layer["type"]]
        subs = [("1", lambda h: mixer(h, mix, layer["mixer"], eps))]
        if layer.get("mlp"):
            subs.append(("2", lambda h: relu2_mlp(h, _sub(weights, f"l{i}.mlp.", dtype))))
        for n, f in subs:
            hc = _sub(weights, f"l{i}.hc{n}.", dtype)
            y = f(rms(hyper_read(xs, hc["in"]), w(f"l{i}.norm{n}"), eps))
            xs = hyper_write(xs, hc["mix"], hc["out"], y)
        if trace is not None:
            trace.append(xs.sum(dim=0))
    return softcap(rms(xs.sum(dim=0), w("final.norm"), eps) @ w("head").T, config["logit_softcap"])


def logits(config, weights, tokens, dtype=torch.float64, trace=None):
    """Of the design that the configuration names."""
    return {"Gafulix": gafulix_logits, "Roletar": roletar_logits}[config["architecture"]](config, weights, tokens, dtype, trace)
