"""HybridEngine against the plain oracle: prompts, portions, decoding, batches, recycled blocks and slots, scheduling,
and the trace runner.  The fp32 engine must agree to fp32 rounding; the bf16 engine to bf16 rounding."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

from hybrid_cases import CONFIGS, logit_error, random_weights, tokens, write_checkpoint
from nanoquantization_amd.engine import HybridEngine, Portion
from nanoquantization_amd.utils.loader import model_from_config
from oracle import hybrid_oracle as o

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
TOL = {torch.float32: 1e-4, torch.bfloat16: 0.15}
_cache = {}      # models and their weights; kept, so that an id names one set of weights


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    def get(name, dtype):
        if (name, dtype) not in _cache:
            path = tmp_path_factory.mktemp(name)
            w = random_weights(CONFIGS[name], rank=12, clear_routing=dtype == torch.bfloat16)
            write_checkpoint(path, CONFIGS[name], w)
            _cache[name, dtype] = model_from_config(str(path), "cuda", dtype), path, w
        return _cache[name, dtype]
    return get


_oracle = {}


def expected(name, weights, ids):
    key = (name, id(weights), tuple(ids))
    if key not in _oracle:
        _oracle[key] = o.logits(CONFIGS[name], weights, ids)
    return _oracle[key]


def run(eng, ids, cuts, lease=None):
    """Logits of every position: portions of the given sizes, the rest one by one through the decode step."""
    own = lease is None
    lease = lease or eng.acquire(0)
    out, at = [], 0
    for n in cuts:
        n = min(n, len(ids) - at)
        if n > 0:
            eng.grow(lease, at + n)
            out.append(eng.extend([Portion(lease, at, ids[at:at + n], list(range(n)))]).clone())
            at += n
    while at < len(ids):
        eng.grow(lease, at + 1)
        out.append(eng.decode([(lease, at, ids[at])]).float().clone())
        at += 1
    if own:
        eng.release(lease)
    return torch.cat(out)


def free_of(eng):
    return sorted(eng.cache.free), sorted(eng.states.free) if eng.states is not None else None


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_prompt_portions_and_decoding_against_oracle(models, name, dtype):
    model, _, w = models(name, dtype)
    V, T = CONFIGS[name]["vocab"], 71
    ids = tokens(T, V, seed=3)
    want = expected(name, w, ids)
    eng = HybridEngine(model, max_batch=1, max_seq_len=128, block_size=16)
    free = free_of(eng)
    for cuts in ([T], [1], [40], [2] * 36, [3, 2, 16, 1, 7, 2, 30], [19, 1, 1, 20, 2]):
        print(f"{name} {dtype} cuts {cuts[:4]}", flush=True)
        got = run(eng, ids, cuts)
        assert logit_error(got, want) <= TOL[dtype], (name, dtype, cuts[:4], logit_error(got, want))
    assert free_of(eng) == free


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("name", [n for n in sorted(CONFIGS) if n.startswith("roletar")])
def test_latent_passes_of_every_form_agree(models, name, dtype):
    """The same portions with their latents expanded, and absorbed into the queries: all of the prompt in one pass, and the
    second half after the first."""
    model, _, w = models(name, dtype)
    ids = tokens(71, CONFIGS[name]["vocab"], seed=3)
    want = expected(name, w, ids)
    for limit in (0, 10 ** 6):
        eng = HybridEngine(model, max_batch=1, max_seq_len=128, block_size=16)
        eng.absorb_rows = limit
        for cuts in ([71], [30, 2, 39]):
            print(f"{name} {dtype} absorbing up to {limit} rows, cuts {cuts}", flush=True)
            assert logit_error(run(eng, ids, cuts), want) <= TOL[dtype], (name, dtype, limit, cuts)


def test_residual_stream_after_every_layer(models):
    for name in sorted(CONFIGS):
        model, _, w = models(name, torch.float32)
        ids = tokens(23, CONFIGS[name]["vocab"], seed=4)
        eng = HybridEngine(model, 1, 64, 16)
        lease, got, want = eng.acquire(2), [], []
        print(f"{name} layer trace", flush=True)
        a = eng.extend([Portion(lease, 0, ids, [22])], trace=got).clone()
        assert torch.allclose(a, eng.extend([Portion(lease, 0, ids, [22])]), atol=1e-5)     # tracing changes nothing
        o.logits(CONFIGS[name], w, ids, trace=want)
        assert len(got) == len(want) == len(eng.runs)
        for g, e in zip(got, want):
            assert (g.double().cpu() - e).abs().max() <= 2e-5 * e.abs().max()


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("name", ["loop_middle", "roletar_loop_middle", "roletar_wide"])
def test_unequal_requests_in_one_batch_equal_each_alone(models, name, dtype):
    model, _, w = models(name, dtype)
    V = CONFIGS[name]["vocab"]
    lens, steps = [1, 45, 20, 33, 2], 6
    seqs = [tokens(n + steps, V, seed=10 + n) for n in lens]
    eng = HybridEngine(model, max_batch=6, max_seq_len=64, block_size=16)
    leases = [eng.acquire(4) for _ in lens]
    # first a pass over uneven beginnings of all of them, then one over the rest together, then decoding as a batch
    cut = [max(1, n // 2) for n in lens]
    got = [[] for _ in lens]
    print(f"batch {dtype}", flush=True)
    for lo, hi in ((lambda i: 0, lambda i: cut[i]), (lambda i: cut[i], lambda i: lens[i])):
        ps = [Portion(leases[i], lo(i), seqs[i][lo(i):hi(i)], list(range(hi(i) - lo(i)))) for i in (3, 0, 4, 1, 2) if hi(i) > lo(i)]
        logits, at = eng.extend(ps), 0
        for p in ps:
            i = leases.index(p.lease)
            got[i].append(logits[at:at + len(p.want)].clone())
            at += len(p.want)
    for s in range(steps):
        logits = eng.decode([(leases[i], lens[i] + s, seqs[i][lens[i] + s]) for i in (4, 2, 0, 1, 3)])
        for r, i in enumerate((4, 2, 0, 1, 3)):
            got[i].append(logits[r:r + 1].clone())
    for i in range(len(lens)):
        assert logit_error(torch.cat(got[i]), expected(name, w, seqs[i])) <= TOL[dtype], (dtype, lens[i])
    for l in leases:
        eng.release(l)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("name", ["no_loop", "roletar_one_stream", "roletar_many"])
def test_blocks_and_slots_used_again(models, name, dtype):
    """One sequence's worth of blocks and one slot, handed from request to request in a different order every time."""
    model, _, w = models(name, dtype)
    V = CONFIGS[name]["vocab"]
    eng = HybridEngine(model, max_batch=1, max_seq_len=64, block_size=16, num_blocks=4, num_slots=1)
    for i, (n, cuts) in enumerate([(60, [30]), (3, [3]), (50, [2] * 25), (1, [1]), (64, [64]), (37, [5])]):
        ids = tokens(n, V, seed=50 + i)
        print(f"reuse {i} {dtype}", flush=True)
        assert logit_error(run(eng, ids, cuts), expected(name, w, ids)) <= TOL[dtype], i
        eng.cache.free = eng.cache.free[1:] + eng.cache.free[:1]
    a = eng.acquire(4)
    with pytest.raises(RuntimeError):
        eng.acquire(0)                       # no slot left
    eng.release(a)


@pytest.mark.parametrize("name", ["loop_all", "roletar_loop_middle"])
def test_long_decoding_stays_on_the_oracle(models, name):
    """Every chunk edge, window, block border and wrap is passed by single decoded tokens."""
    for dtype in (torch.float32, torch.bfloat16):
        model, _, w = models(name, dtype)
        ids = tokens(150, CONFIGS[name]["vocab"], seed=8)
        eng = HybridEngine(model, max_batch=1, max_seq_len=192, block_size=16)
        print(f"long decoding {dtype}", flush=True)
        assert logit_error(run(eng, ids, [1]), expected(name, w, ids)) <= TOL[dtype]


@pytest.mark.parametrize("name", ["loop_middle", "roletar_loop_middle"])
def test_graph_replays_equal_eager_steps(models, name):
    model, _, _ = models(name, torch.bfloat16)
    ids = tokens(40, CONFIGS[name]["vocab"], seed=9)
    outs = []
    for graph in (False, True):
        print(f"graph={graph}", flush=True)
        eng = HybridEngine(model, max_batch=3, max_seq_len=64, block_size=16, use_graph=graph)
        lease, rows = eng.acquire(4), []
        eng.extend([Portion(lease, 0, ids[:10], [])])
        for t in range(10, 40):
            rows.append(eng.decode([(lease, t, ids[t])]).clone())
            if t % 7 == 0:                  # eager work of the same kind between the replays
                other = eng.acquire(1)
                eng.extend([Portion(other, 0, ids[:5], [4])])
                eng.release(other)
                torch.cuda.synchronize()
        assert (eng._graph is not None) == graph
        outs.append(torch.cat(rows))
    assert torch.equal(outs[0], outs[1])


@pytest.mark.parametrize("name", ["loop_all", "roletar_loop_middle"])
@pytest.mark.parametrize("rows", [20, 40, 70])
def test_wider_batches_with_and_without_graph(models, rows, name):
    """Enough rows for the other forms of the linears and experts (and, at 70, for the library's products, which stay out
    of a graph): the same tokens from graph replays and from eager steps, for unequal requests that come and go."""
    model, _, _ = models(name, torch.bfloat16)
    V = CONFIGS[name]["vocab"]
    reqs = [(tokens(1 + (7 * i) % 23, V, seed=200 + i), 3 + i % 9) for i in range(rows + 7)]
    outs = []
    for graph in (False, True, True):
        print(f"{rows} rows graph={graph}", flush=True)
        eng = HybridEngine(model, max_batch=rows, max_seq_len=48, block_size=16, use_graph=graph)
        outs.append(eng.serve(reqs))
        assert (eng._graph is not None) == (graph and rows <= 64)
        assert eng.serve(reqs) == outs[-1]          # the captured graph again, rows and slots dealt anew
    assert outs[0] == outs[1] == outs[2] and [len(t) for t in outs[0]] == [n for _, n in reqs]


def greedy_reference(name, weights, prompt, new):
    seq, gaps = list(prompt), []
    for _ in range(new):
        top = o.logits(CONFIGS[name], weights, seq)[-1].topk(2)
        gaps.append((top.values[0] - top.values[1]).item())
        seq.append(top.indices[0].item())
    return seq[len(prompt):], gaps


@pytest.mark.parametrize("name", ["one_pass_loop", "roletar_loop_middle"])
def test_generate_and_serve_greedy(models, name):
    """Through the schedulers: the fp32 engine picks the oracle's tokens; requests of any lengths, rows, blocks and slots
    recycled, long prompts in portions."""
    new = 8
    model, _, w = models(name, torch.float32)
    V = CONFIGS[name]["vocab"]
    prompts = [tokens(n, V, seed=70 + n) for n in (19, 19, 19)]
    refs = [greedy_reference(name, w, p, new) for p in prompts]
    eng = HybridEngine(model, max_batch=4, max_seq_len=96, block_size=16)
    print("generate fp32", flush=True)
    got = eng.generate(prompts, new)
    for g, (ref, gaps) in zip(got, refs):
        clear = next((i for i, d in enumerate(gaps) if d < 1e-3), new)
        assert clear > new // 2 and g[:clear] == ref[:clear]
    lens = [1, 40, 7, 66, 19, 2, 33]
    reqs = [(tokens(n, V, seed=90 + n), 3 + n % 6) for n in lens]
    for dtype in (torch.float32, torch.bfloat16):
        model, _, _ = models(name, dtype)
        alone = HybridEngine(model, max_batch=1, max_seq_len=96, block_size=16)
        want = [alone.serve([r])[0] for r in reqs]
        for kw in (dict(), dict(batch_prefill=True), dict(batch_prefill=True, max_prefill_tokens=50)):
            print(f"serve {dtype} {kw}", flush=True)
            eng = HybridEngine(model, max_batch=3, max_seq_len=96, block_size=16, num_blocks=14, prefill_tokens=25)
            free = (sorted(eng.cache.free), sorted(eng.states.free))
            st = {}
            got = eng.serve(reqs, stats=st, **kw)
            assert (sorted(eng.cache.free), sorted(eng.states.free)) == free and st["prefills"] == len(reqs)
            assert [len(g) for g in got] == [m for _, m in reqs]
            same = sum(a == b for a, b in zip(got, want))
            # fp32: rounding alone separates batched from single runs; bf16 may flip a near-tie
            assert same == len(reqs) if dtype == torch.float32 else same >= len(reqs) - 2, (dtype, kw, same)
    eos = want[1][2]
    eng = HybridEngine(model, max_batch=3, max_seq_len=96, block_size=16)
    cut = eng.serve(reqs[:3], eos_token_id=eos)
    assert all(eos not in c[:-1] for c in cut)


@pytest.mark.parametrize("name", ["no_loop", "roletar_one_stream"])
def test_command_line_generates(models, tmp_path, name):
    _, path, _ = models(name, torch.bfloat16)
    cmd = [sys.executable, "-m", "nanoquantization_amd.generate", "--model", str(path), "--max-new-tokens", "5",
           "--prompt-ids", "3,1,4", "--prompt-ids", "15,9,2,6"]
    print("cli", flush=True)
    r = subprocess.run(cmd, cwd=ROOT, stdout=subprocess.PIPE, stderr=subprocess.PIPE, text=True, timeout=110)
    assert r.returncode == 0, r.stderr[-2000:]
    lines = [json.loads(l) for l in r.stdout.splitlines() if l.startswith("{")]
    assert [l["prompt"] for l in lines] == [[3, 1, 4], [15, 9, 2, 6]] and all(len(l["tokens"]) == 5 for l in lines)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["loop_middle", "roletar_loop_middle"])
def test_trace_runner(models, tmp_path, name, dtype):
    _, path, w = models(name, torch.bfloat16)
    V = CONFIGS[name]["vocab"]
    a, b = tokens(40, V, seed=21), tokens(9, V, seed=22)
    steps = [dict(step=0, entries=[dict(id="x", tokens=a[:17], want=[0, 16])], end=[]),
             dict(step=1, entries=[dict(id="x", tokens=a[17:19], want=[])], end=[]),
             dict(step=2, entries=[dict(id="x", tokens=a[19:20], want=[0]), dict(id="y", tokens=b[:1], want=[0])], end=[]),
             dict(step=3, entries=[dict(id="y", tokens=b[1:], want=[7]), dict(id="x", tokens=a[20:], want=[19, 3])], end=["x", "y"]),
             dict(step=4, entries=[dict(id="x", tokens=b[:4], want=[3])], end=["x"])]
    print(f"trace runner {dtype}", flush=True)
    r = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", str(path), "--dtype", dtype, "--out", str(tmp_path),
                        "--max-tokens", "64"], input="".join(json.dumps(s) + "\n" for s in steps), stdout=subprocess.PIPE,
                       stderr=subprocess.PIPE, text=True, timeout=110)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [l for l in r.stdout.splitlines() if l.startswith("done")] == [f"done {i}" for i in range(5)]
    ea, eb = expected(name, w, a), expected(name, w, b)
    want = {0: ea[[0, 16]], 2: torch.stack([ea[19], eb[0]]), 3: torch.stack([eb[8], ea[39], ea[23]]), 4: eb[3:4]}
    assert sorted(os.listdir(tmp_path)) == [f"{i}.f32" for i in sorted(want)]
    for i, e in want.items():
        got = torch.from_numpy(np.fromfile(tmp_path / f"{i}.f32", dtype="<f4").reshape(-1, V))
        d = got.double() - e
        d = d - d.mean(-1, keepdim=True)
        assert (d.pow(2).mean(-1).sqrt() / e.std()).max() <= TOL[getattr(torch, dtype)], i
