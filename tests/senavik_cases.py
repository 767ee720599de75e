"""Scenarios for the Senavik family, run by the CPU tests (reference ops,
fp32) and the GPU tests (HIP kernels, fp32 and bf16). Every scenario builds
a small configuration with random weights, runs it through the engine and
compares with the plain model in senavik_oracle.py."""
import copy

import torch

import senavik_oracle as oracle
from bezizen_cases import _act, _close, _maps, portions, row_errors, tokens
from kukeon_amd.engine.config import EngineConfig, SamplingParams
from kukeon_amd.engine.engine import LLMEngine
from kukeon_amd.engine.kv_cache import SequenceKV
from kukeon_amd.models.feedforward import RoutedMoE
from kukeon_amd.models.rotary import angle_table
from kukeon_amd.models.senavik import SenavikConfig, SenavikModel


def banded(factor=6.0, low=1.5, high=4.0, original=60):
    return {"factor": factor, "low": low, "high": high, "original": original}


def yarn(factor=3.0, original=80, fast=6.0, slow=1.0):
    return {"factor": factor, "original": original, "fast": fast,
            "slow": slow}


def attn(heads=4, kv_heads=2, dim=10, vdim=7, rot=6, base=30.0,
         scaling=banded(), window=9, keep=3, scale=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
         "rot": {"base": base, "dims": rot},
         "scale": scale if scale is not None else 1.5 * dim ** -0.5}
    if scaling:
        m["rot"]["scaling"] = scaling
    if window:
        m["mask"] = {"size": window, "keep_first": keep}
    return {"type": "attention", "mixer": m}


def latent(heads=3, dim=5, rot_dim=6, vdim=9, q_rank=11, kv_rank=13,
           base=25.0, scaling=yarn(), scale=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim,
         "q_rank": q_rank, "kv_rank": kv_rank,
         "rot": {"base": base, "dims": rot_dim},
         "scale": scale if scale is not None else
         1.2 * (dim + rot_dim) ** -0.5}
    if scaling:
        m["rot"]["scaling"] = scaling
    return {"type": "latent_attention", "mixer": m}


def moe(experts, top, ff, groups=None):
    r = {"experts": experts, "top": top}
    if groups:
        r["groups"] = {"count": groups[0], "keep": groups[1]}
    return {"kind": "moe", "expert": {"ff": ff}, "router": r}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def layer(mix, mlp):
    return dict(mix, mlp=mlp)


def config(layers, width=40, vocab=45, eps=1e-4):
    return {"architecture": "Senavik", "width": width, "vocab": vocab,
            "norm": {"eps": eps}, "layers": layers}


CONFIGS = {
    # both mixers, all feed-forwards and none, sizes off every vector path
    "hybrid": lambda: config([
        layer(attn(), moe(6, 2, 9, (3, 2))),
        layer(latent(), dense(21)),
        layer(attn(heads=3, kv_heads=3, dim=6, vdim=11, rot=2, base=7.0,
                   window=5, keep=1), None),
        layer(latent(heads=2, dim=4, rot_dim=2, vdim=3, kv_rank=20), moe(
            8, 3, 10, (4, 3))),
        layer(attn(heads=6, kv_heads=2, dim=8, vdim=5, rot=8, window=14,
                   keep=6), moe(5, 2, 7)),
    ]),
    # rows of whole 16-byte pieces (the vector forms), a rotated part that
    # ends inside one, four query heads on one kv head
    "aligned": lambda: config([
        layer(attn(heads=4, kv_heads=1, dim=40, vdim=24, rot=20, window=20,
                   keep=2), moe(8, 2, 64, (2, 1))),
        layer(latent(heads=4, dim=24, rot_dim=16, vdim=16, q_rank=48,
                     kv_rank=64), dense(72)),
        layer(attn(heads=2, kv_heads=2, dim=96, vdim=48, rot=32, window=31,
                   keep=4), moe(16, 4, 32, (4, 2))),
    ], width=128, vocab=50, eps=1e-3),
    # everything at its simplest: no scaling, no window, no groups, one head,
    # one expert, a width off multiples of 8
    "plain": lambda: config([
        layer(attn(heads=1, kv_heads=1, dim=7, vdim=1, rot=4, scaling=None,
                   window=0), moe(1, 1, 5)),
        layer(latent(heads=1, dim=3, rot_dim=2, vdim=2, q_rank=5, kv_rank=4,
                     scaling=None), None),
        layer(attn(heads=2, kv_heads=1, dim=4, vdim=9, rot=0, scaling=None,
                   window=6, keep=0), dense(9)),
    ], width=26, vocab=31),
    # a window of the token itself, groups of one expert, all experts chosen
    "extreme": lambda: config([
        layer(attn(heads=2, kv_heads=1, dim=8, vdim=8, rot=8, window=1,
                   keep=1), moe(4, 3, 8, (4, 3))),
        layer(attn(heads=2, kv_heads=2, dim=8, vdim=16, rot=2, window=2,
                   keep=40), moe(3, 3, 8)),
        layer(latent(heads=5, dim=2, rot_dim=4, vdim=8, q_rank=3, kv_rank=8),
              moe(6, 4, 8, (2, 2))),
    ], width=16, vocab=21, eps=1e-2),
    "only_latent": lambda: config([
        layer(latent(heads=2, dim=8, rot_dim=8, vdim=8, q_rank=16,
                     kv_rank=300), None),
        layer(latent(heads=3, dim=1, rot_dim=2, vdim=4), dense(8)),
    ], width=16, vocab=21),
    "only_attention": lambda: config([
        layer(attn(heads=2, kv_heads=2, dim=8, vdim=8, window=300, keep=2),
              None),
        layer(attn(heads=3, kv_heads=1, dim=8, vdim=16, window=4, keep=0),
              moe(3, 2, 8)),
    ], width=16, vocab=21),
    # heads of 128 on pages of 16, a latent of 128 with a rotated part of 32:
    # the sizes of the matrix-core kernels; a window that ends inside a key
    # tile, three query heads per kv head, more kept tokens than one tile
    "tiles": lambda: config([
        layer(attn(heads=6, kv_heads=2, dim=128, vdim=128, rot=64, window=40,
                   keep=5, scale=0.12), moe(4, 2, 16, (2, 1))),
        layer(latent(heads=4, dim=16, rot_dim=32, vdim=8, q_rank=16,
                     kv_rank=128, scale=0.1), None),
        layer(attn(heads=3, kv_heads=1, dim=128, vdim=128, rot=128, window=33,
                   keep=37, scale=0.1), dense(24)),
    ], width=48, vocab=40),
    # a window longer than one pass of the row kernel over the keys, and more
    # kept tokens than one of its key tiles
    "long_window": lambda: config([
        layer(attn(heads=2, kv_heads=1, dim=8, vdim=8, window=150, keep=70,
                   scale=0.9), None),
        layer(latent(heads=2, dim=8, rot_dim=8, vdim=8, kv_rank=16),
              moe(4, 2, 8, (2, 1))),
    ], width=16, vocab=19),
}


def weights(cfg, seed=0):
    """Random checkpoint for a config dictionary, bf16 like a stored one."""
    g = torch.Generator().manual_seed(seed)
    W, V = cfg["width"], cfg["vocab"]

    def r(*shape, std=1.0, mean=0.0):
        return (torch.randn(*shape, generator=g) * std + mean).to(
            torch.bfloat16)

    t = {"embed": r(V, W, std=0.3), "embed.norm": r(W, std=0.3),
         "final.norm": r(W, std=0.3), "head": r(V, W, std=W ** -0.5)}
    for i, L in enumerate(cfg["layers"]):
        p = "l%d." % i
        m = L["mixer"]
        t[p + "norm1"] = r(W, std=0.3)
        q = p + "mix."
        H, D, U = m["heads"], m["dim"], m["vdim"]
        t[q + "sink"] = r(H, std=1.0, mean=1.0)
        t[q + "o"] = r(W, H * U, std=1.5 * (H * U) ** -0.5)
        if L["type"] == "attention":
            G = m["kv_heads"]
            t[q + "q"] = r(H * D, W, std=1.3 * W ** -0.5)
            t[q + "k"] = r(G * D, W, std=1.3 * W ** -0.5)
            t[q + "v"] = r(G * U, W, std=W ** -0.5)
        else:
            R, Q, C = m["rot_dim"], m["q_rank"], m["kv_rank"]
            t[q + "dq"] = r(Q, W, std=W ** -0.5)
            t[q + "dq.norm"] = r(Q, std=0.3, mean=1.0)
            t[q + "uq"] = r(H * (D + R), Q, std=Q ** -0.5)
            t[q + "dkv"] = r(C + R, W, std=W ** -0.5)
            t[q + "dkv.norm"] = r(C, std=0.3, mean=1.0)
            t[q + "uk"] = r(H * D, C, std=C ** -0.5)
            t[q + "uv"] = r(H * U, C, std=C ** -0.5)
        f = L["mlp"]
        if not f:
            continue
        t[p + "norm2"] = r(W, std=0.3)
        q = p + "mlp."
        if f["kind"] == "dense":
            t[q + "up"] = r(f["ff"], W, std=W ** -0.5)
            t[q + "down"] = r(W, f["ff"], std=f["ff"] ** -0.5)
            continue
        E, ff = f["router"]["experts"], f["expert"]["ff"]
        t[q + "router"] = r(E, W, std=2.0 * W ** -0.5)
        t[q + "correction"] = r(E, std=0.3, mean=-0.4)
        for e in range(E):
            t[q + f"e{e}.gate"] = r(ff, W, std=1.2 * W ** -0.5)
            t[q + f"e{e}.up"] = r(ff, W, std=1.2 * W ** -0.5)
            t[q + f"e{e}.down"] = r(W, ff, std=ff ** -0.5)
    return t


def poison(eng):
    """What a sequence has not written itself must never be read."""
    for t in list(eng.kv.k) + list(eng.kv.v):
        if t is not None and t.numel():
            t.fill_(300.0)


def make_engine(cfg, tensors, device, dtype, blocks=96, slots=4,
                block_size=4, max_len=384, dirty=True, **ekw):
    mcfg = SenavikConfig.from_json(cfg)
    model = SenavikModel(mcfg, device=device, dtype=dtype, tensors=tensors,
                         max_position=max_len)
    kw = dict(block_size=block_size, max_model_len=max_len,
              max_sessions=slots, num_kv_blocks=blocks, use_graphs=False)
    kw.update(ekw)
    eng = LLMEngine(model, mcfg, EngineConfig(**kw), device=device)
    if dirty:
        poison(eng)
    return eng


def logits_of(cfg, W, toks, got=None):
    """The plain model's logits; with `got`, a run's result, under the
    experts that the run chose."""
    return oracle.forward(toks, W, cfg,
                          choices=None if got is None else got.choices)


def tol(dtype):
    return 2e-4 if dtype == "fp32" else 0.1


def check(got, want, dtype, what=""):
    """fp32: every row within the tolerance. bf16: half of the rows within
    two fifths of it, nine in ten (all but one of a few) within it, none far
    off; small widths make single rows round badly."""
    e = row_errors(got, want)
    over = int((e > tol(dtype)).sum())
    if dtype == "fp32":
        assert over == 0, f"{what}: error {float(e.max()):.3g}"
        return
    assert float(e.median()) <= 0.4 * tol(dtype), \
        f"{what}: median {float(e.median()):.3g}"
    assert over <= max(1, e.numel() // 10) and float(e.max()) <= 0.5, \
        f"{what}: {over} rows over {tol(dtype)}, worst {float(e.max()):.3g}"


class Routes:
    """Records what the engine's routers chose, call by call."""

    def __init__(self, eng):
        self.mods = [L.ff for L in eng.model.layers
                     if isinstance(L.ff, RoutedMoE)]

    def __enter__(self):
        self.seen = []
        for m in self.mods:
            def rec(idx, wts, logits, m=m, fn=m._route):
                fn(idx, wts, logits)
                self.seen.append(idx[:, :m.f.top].cpu().long().clone())
            m._route = rec
        return self

    def __exit__(self, *exc):
        for m in self.mods:
            del m._route


def run_schedule(eng, prompts, schedule):
    """schedule: list of steps, each a list of (request index, count).
    -> per request the logits at every position [len, vocab], with the
    experts chosen on the way as their `choices`. A request is freed when it
    is through."""
    kvs, at = {}, {}
    out = {i: [] for i in range(len(prompts))}
    picks = {i: [] for i in range(len(prompts))}
    for step in schedule:
        entries, want = [], []
        for i, n in step:
            if i not in kvs:
                kvs[i] = SequenceKV(eng.ecfg.block_size)
                at[i] = 0
            entries.append((kvs[i], prompts[i][at[i]: at[i] + n]))
            want.append(list(range(n)))
        with Routes(eng) as routes:
            lg = eng.forward_tokens(entries, want)
        row = 0
        for i, n in step:
            out[i].append(lg[row: row + n])
            picks[i].append([c[row: row + n] for c in routes.seen])
            row += n
            at[i] += n
            if at[i] == len(prompts[i]):
                eng.free_sequence(kvs.pop(i))
    res = {}
    for i, v in out.items():
        if v:
            res[i] = torch.cat(v)
            res[i].choices = [torch.cat(c) for c in zip(*picks[i])]
    return res


def same_choices(a, b):
    return all(torch.equal(x.sort(-1).values, y.sort(-1).values)
               for x, y in zip(a.choices, b.choices))


# ---------------------------------------------------------------- scenarios
def case_whole(name, device, dtype, n=27):
    cfg = CONFIGS[name]()
    W = weights(cfg, 1)
    toks = tokens(cfg, n, 1)
    eng = make_engine(cfg, W, device, dtype,
                      block_size=16 if name == "tiles" else 4)
    got = run_schedule(eng, [toks], [[(0, len(toks))]])[0]
    check(got, logits_of(cfg, W, toks, got), dtype, name)


def case_layers(device, dtype):
    """The residual stream after every layer."""
    cfg = CONFIGS["hybrid"]()
    W = weights(cfg, 2)
    toks = tokens(cfg, 17, 2)
    eng = make_engine(cfg, W, device, dtype)
    kv = SequenceKV(eng.ecfg.block_size)
    got, want = [], []
    fwd = eng.model.forward
    eng.model.forward = lambda *a, **k: fwd(*a, taps=got, **k)
    with Routes(eng) as routes:
        eng.forward_tokens([(kv, toks)])
    eng.model.forward = fwd
    oracle.forward(toks, W, cfg, want, routes.seen)
    assert len(got) == len(want) == len(cfg["layers"])
    for i, (g, w) in enumerate(zip(got, want)):
        e = row_errors(g, w)
        over = int((e > tol(dtype)).sum())
        assert over <= (0 if dtype == "fp32" else 1), \
            f"layer {i}: {float(e.max()):.3g}"


def case_prefill_vs_decode(name, device, dtype):
    cfg = CONFIGS[name]()
    W = weights(cfg, 3)
    toks = tokens(cfg, 25, 3)
    whole = run_schedule(make_engine(cfg, W, device, dtype), [toks],
                         [[(0, len(toks))]])[0]
    one = run_schedule(make_engine(cfg, W, device, dtype), [toks],
                       [[(0, 1)] for _ in toks])[0]
    check(whole, logits_of(cfg, W, toks, whole), dtype, "whole")
    check(one, logits_of(cfg, W, toks, one), dtype, "token by token")
    if same_choices(one, whole):
        check(one, whole, dtype, "token by token against whole")


def case_portions(name, device, dtype, sizes, n=41):
    cfg = CONFIGS[name]()
    W = weights(cfg, 4)
    toks = tokens(cfg, n, 4)
    sched = [[(0, k)] for k in portions(len(toks), sizes)]
    got = run_schedule(make_engine(cfg, W, device, dtype), [toks], sched)[0]
    check(got, logits_of(cfg, W, toks, got), dtype, f"portions {sizes}")


def case_batch(name, device, dtype):
    """Unequal requests in one batch, portions beside single tokens."""
    cfg = CONFIGS[name]()
    W = weights(cfg, 5)
    prompts = [tokens(cfg, n, 10 + n) for n in (19, 1, 7, 30)]
    sched = [
        [(0, 5), (1, 1), (3, 2)],
        [(0, 1), (2, 7), (3, 9)],
        [(3, 1), (0, 1)],
        [(0, 12), (3, 1)],
        [(3, 17)],
    ]
    got = run_schedule(make_engine(cfg, W, device, dtype), prompts, sched)
    for i, p in enumerate(prompts):
        alone = run_schedule(make_engine(cfg, W, device, dtype), [p],
                             [[(0, len(p))]])[0]
        check(got[i], logits_of(cfg, W, p, got[i]), dtype, f"request {i}")
        if same_choices(got[i], alone):
            check(got[i], alone, dtype, f"request {i} against itself alone")


def case_reuse(device, dtype):
    """A pool too small for all requests at once: pages of finished requests
    are handed to the next ones."""
    cfg = CONFIGS["hybrid"]()
    W = weights(cfg, 6)
    prompts = [tokens(cfg, n, 20 + n) for n in (14, 11, 16, 3, 13)]
    eng = make_engine(cfg, W, device, dtype, blocks=8, slots=2, block_size=4)
    sched = [
        [(0, 6), (1, 4)],
        [(0, 8), (1, 1)],          # 0 ends: 4 pages come back
        [(1, 6), (2, 9)],          # 1 ends
        [(2, 7), (3, 2)],          # 2 ends
        [(3, 1), (4, 12)],         # 3 ends
        [(4, 1)],
    ]
    got = run_schedule(eng, prompts, sched)
    for i, p in enumerate(prompts):
        check(got[i], logits_of(cfg, W, p, got[i]), dtype, f"request {i}")
    assert eng.kv.allocator.num_free == 8


def case_first_tokens(device, dtype):
    """Short sequences started in used pages, and a start cut into single
    tokens."""
    for name in ("hybrid", "extreme"):
        cfg = CONFIGS[name]()
        W = weights(cfg, 7)
        eng = make_engine(cfg, W, device, dtype, slots=1)
        for n, sched in ((1, [1]), (2, [2]), (3, [1, 2]),
                         (9, [1, 1, 1, 2, 4]), (6, [2, 1, 3])):
            toks = tokens(cfg, n, 30 + n)
            got = run_schedule(eng, [toks], [[(0, k)] for k in sched])[0]
            check(got, logits_of(cfg, W, toks, got), dtype, f"{name} {n}")


def case_long_decode(device, dtype):
    """Decoding past every window and through many pages."""
    cfg = CONFIGS["hybrid"]()
    W = weights(cfg, 8)
    toks = tokens(cfg, 75, 8)
    sched = [[(0, 3)]] + [[(0, 1)] for _ in range(72)]
    got = run_schedule(make_engine(cfg, W, device, dtype, block_size=4),
                       [toks], sched)[0]
    check(got, logits_of(cfg, W, toks, got), dtype, "long decode")


def case_long_window(device, dtype):
    """A window longer than one pass of the row kernel over the keys, kept
    tokens beside it, portions that end inside both."""
    cfg = CONFIGS["long_window"]()
    W = weights(cfg, 9)
    toks = tokens(cfg, 270, 9)
    eng = make_engine(cfg, W, device, dtype, blocks=200, max_len=400)
    sched = [[(0, 69)], [(0, 2)], [(0, 146)], [(0, 20)]] + [[(0, 1)]] * 33
    got = run_schedule(eng, [toks], sched)[0]
    check(got, logits_of(cfg, W, toks, got), dtype, "portions and decoding")
    whole = run_schedule(eng, [toks], [[(0, 270)]])[0]
    if same_choices(whole, got):
        check(whole, got, dtype, "whole")


def case_long_portions(device, dtype):
    """Portions long enough for the matrix-core attention kernel beside
    single tokens, cut inside a window and inside a key tile."""
    cfg = CONFIGS["tiles"]()
    W = weights(cfg, 13)
    prompts = [tokens(cfg, n, 80 + n) for n in (150, 61, 40)]
    eng = make_engine(cfg, W, device, dtype, blocks=40, block_size=16,
                      max_len=256)
    sched = [
        [(0, 70), (1, 20)],
        [(0, 1), (1, 41), (2, 39)],
        [(0, 45), (2, 1)],
        [(0, 34)],
    ]
    got = run_schedule(eng, prompts, sched)
    for i in range(3):
        check(got[i], logits_of(cfg, W, prompts[i], got[i]), dtype,
              f"request {i}")


def case_sorted_experts(device, dtype):
    """Long portions sort their rows by expert and run each expert over its
    rows at once; short steps take the pair kernels."""
    cfg = CONFIGS["hybrid"]()
    W = weights(cfg, 12)
    prompts = [tokens(cfg, n, 70 + n) for n in (80, 70)]
    eng = make_engine(cfg, W, device, dtype, blocks=64, max_len=128)
    got = run_schedule(eng, prompts, [[(0, 80), (1, 69)], [(1, 1)]])
    for i in range(2):
        check(got[i], logits_of(cfg, W, prompts[i], got[i]), dtype,
              f"sorted rows, request {i}")


def case_generate(device, dtype, use_graphs=False):
    """Greedy generation through add_request / step: every token is the plain
    model's best one after the tokens before it, except where the plain
    model's two best logits nearly tie."""
    cfg = CONFIGS["hybrid"]()
    W = weights(cfg, 10)
    prompts = [tokens(cfg, n, 50 + n) for n in (9, 4, 13)]
    new = 10
    eng = make_engine(cfg, W, device, dtype, use_graphs=use_graphs,
                      graph_buckets=(4,), decode_microbatch=4)
    sp = SamplingParams(temperature=0.0, top_k=1, top_p=1.0,
                        max_new_tokens=new)
    kvs = [SequenceKV(eng.ecfg.block_size) for _ in prompts]
    rids = [eng.add_request(kv, p, sp) for kv, p in zip(kvs, prompts)]
    outs = {r: [] for r in rids}
    for _ in range(200):
        if not eng.has_work():
            break
        for o in eng.step():
            outs[o.req_id].extend(o.new_tokens)
    assert not eng.has_work()
    margin = 0.02 if dtype == "fp32" else 0.4
    checked = 0
    for rid, p in zip(rids, prompts):
        got = outs[rid]
        assert len(got) == new
        # one pass over the whole sequence gives every step's logits
        lgs = logits_of(cfg, W, list(p) + got)
        for k in range(new):
            lg = lgs[len(p) + k - 1]
            top2 = lg.topk(2).values
            if float(top2[0] - top2[1]) < margin:
                continue
            assert got[k] == int(lg.argmax()), f"request {rid}, token {k}"
            checked += 1
    assert checked >= (15 if dtype == "fp32" else 3)
    for kv in kvs:
        eng.free_sequence(kv)
    assert eng.kv.allocator.num_free == eng.kv.num_blocks


def case_graph_replays(device, dtype):
    """Steps under captured graphs against the same steps run eagerly."""
    cfg = CONFIGS["aligned"]()
    W = weights(cfg, 17)
    prompts = [tokens(cfg, n, 90 + n) for n in (21, 5)]
    outs = []
    for graphs in (False, True):
        eng = make_engine(cfg, W, device, dtype, use_graphs=graphs,
                          graph_buckets=(4,), decode_microbatch=3)
        got = []
        for turn in range(3):            # eager work between the replays
            kvs = [SequenceKV(eng.ecfg.block_size) for _ in prompts]
            sp = SamplingParams(temperature=0.0, top_k=1, top_p=1.0,
                                max_new_tokens=10)
            rids = [eng.add_request(kv, p[turn:], sp)
                    for kv, p in zip(kvs, prompts)]
            res = {r: [] for r in rids}
            while eng.has_work():
                for o in eng.step():
                    res[o.req_id].extend(o.new_tokens)
            got += [res[r] for r in rids]
            for kv in kvs:
                eng.free_sequence(kv)
        outs.append(got)
    # graphs pad the batch to a bucket, which may reorder a few sums of the
    # library's products, so late tokens may part after a close call
    same = sum(a[k] == b[k] for a, b in zip(*outs) for k in range(10))
    assert same >= 0.8 * 10 * len(outs[0]), f"{same} of {10 * len(outs[0])}"
    assert all(a[0] == b[0] for a, b in zip(*outs))


def assert_greedy(cfg, W, prompt, got, what=""):
    """Every generated token is the plain model's best one, up to the
    rounding of the logits to bfloat16 that the sampler works on."""
    lgs = logits_of(cfg, W, list(prompt) + list(got))
    for i, t in enumerate(got):
        lg = lgs[len(prompt) + i - 1]
        best = float(lg.max())
        assert float(lg[t]) >= best - abs(best) * 2.0 ** -7, \
            f"{what}: token {i} is {t}, the plain model says " \
            f"{int(lg.argmax())}"


def _generate(eng, kv, prompt, n):
    sp = SamplingParams(temperature=0.0, max_new_tokens=n)
    eng.add_request(kv, prompt, sp)
    out = []
    while eng.has_work():
        for o in eng.step():
            out.extend(o.new_tokens)
    return out


def case_multi_turn(device):
    """A session's second turn continues from its pages; an idle session
    whose pages were taken away is rebuilt from its history."""
    cfg = CONFIGS["hybrid"]()
    W = weights(cfg, 15)
    eng = make_engine(cfg, W, device, "fp32", blocks=12, slots=2, max_len=64,
                      dirty=False, decode_microbatch=2)
    a, b = SequenceKV(4), SequenceKV(4)
    p1, p2, p3 = tokens(cfg, 9, 60), tokens(cfg, 5, 61), tokens(cfg, 30, 62)
    t1 = _generate(eng, a, p1, 4)
    assert_greedy(cfg, W, p1, t1, "first turn")
    t2 = _generate(eng, a, p2, 3)
    assert_greedy(cfg, W, p1 + t1 + p2, t2, "second turn")
    assert a.num_tokens > 0
    tb = _generate(eng, b, p3, 4)       # needs a's pages
    assert_greedy(cfg, W, p3, tb, "other session")
    assert a.num_tokens == 0 and a.history
    eng.free_sequence(b)
    t3 = _generate(eng, a, [7, 3], 3)
    assert_greedy(cfg, W, p1 + t1 + p2 + t2 + [7, 3], t3, "rebuilt session")


# ----------------------------------------------------- mechanisms, one by one
def _b(t):
    return t.to(torch.bfloat16)


def pointing(kind, strength=12.0, window=0, keep=0, dim=20, vdim=8):
    """A one-layer stack whose token 8 a + b asks for keys of kind a and is
    itself a key of kind b; norms are neutral and the rotated entries empty,
    so a score is `strength` where the kinds meet and 0 elsewhere. The values
    are the keys' kinds."""
    Wd, V, H = 16, 64, 2
    if kind == "attention":
        mix = attn(heads=H, kv_heads=1, dim=dim, vdim=vdim, rot=4,
                   window=window, keep=keep, scale=strength / 8.0)
    else:
        # latent rows: one entry of `rank`, sqrt(rank) after their norm; the
        # query latent has 8 entries, sqrt(8) after its norm
        rank = 128 if dim == 128 else 16
        mix = latent(heads=H, dim=8, rot_dim=32 if dim == 128 else 4,
                     vdim=vdim, q_rank=8, kv_rank=rank,
                     scale=strength / (8.0 * rank) ** 0.5)
    cfg = config([layer(mix, None)], width=Wd, vocab=V, eps=1e-6)
    W = weights(cfg, 20)
    emb = torch.zeros(V, Wd)
    for v in range(V):
        emb[v, v % 8] = 1.0
        emb[v, 8 + v // 8] = 1.0
    W["embed"] = _b(emb)
    for n in ("embed.norm", "l0.norm1", "final.norm"):
        W[n] = _b(torch.zeros(Wd))
    W["l0.mix.sink"] = _b(torch.tensor([0.0, 2.0]))
    eye = torch.eye(8)
    if kind == "attention":
        wq, wk = torch.zeros(H, dim, Wd), torch.zeros(dim, Wd)
        wq[:, 4:12, 8:] = eye
        wk[4:12, :8] = eye
        wv = torch.zeros(vdim, Wd)
        wv[:8, :8] = eye
        W["l0.mix.q"] = _b(wq.view(-1, Wd))
        W["l0.mix.k"], W["l0.mix.v"] = _b(wk), _b(wv)
    else:
        m = mix["mixer"]
        R, C = m["rot_dim"], m["kv_rank"]
        dq = torch.zeros(8, Wd)
        dq[:, 8:] = eye
        uq = torch.zeros(H, 8 + R, 8)
        uq[:, :8] = eye
        dkv = torch.zeros(C + R, Wd)
        dkv[:8, :8] = eye
        uk, uv = torch.zeros(H, 8, C), torch.zeros(H, vdim, C)
        uk[:, :, :8] = eye
        uv[:, :8, :8] = eye
        W.update({"l0.mix.dq": _b(dq), "l0.mix.dq.norm": _b(torch.ones(8)),
                  "l0.mix.uq": _b(uq.view(-1, 8)), "l0.mix.dkv": _b(dkv),
                  "l0.mix.dkv.norm": _b(torch.ones(C)),
                  "l0.mix.uk": _b(uk.view(-1, C)),
                  "l0.mix.uv": _b(uv.view(-1, C))})
    return cfg, W


def _moved(a, b):
    return float((a - b).abs().max())


def case_window_edges(device, dtype, decode, dim=20, vdim=8, bs=4):
    """One key that every query points at: the first token, the last kept
    and the first not kept one, places at page borders and around the
    window's edge. Just inside the window it is nearly all of the output;
    one place further it is gone, unless it is kept."""
    window, keep = 10, 3
    cfg, W = pointing("attention", window=window, keep=keep, dim=dim,
                      vdim=vdim)
    n = 37
    for target in (0, keep - 1, keep, bs - 1, bs, 2 * bs - 1, 2 * bs, 12,
                   n - window - 1, n - window, n - 1):
        toks = [8 * 1 + 0] * n
        toks[target] = 8 * 1 + 1
        want = logits_of(cfg, W, toks)
        without = logits_of(cfg, W, [8 * 1 + 0] * n)
        for i in range(target + 1, n):
            seen = i - target < window or target < keep
            assert (_moved(want[i], without[i]) > 0.3) == seen
        eng = make_engine(cfg, W, device, dtype, block_size=bs)
        if decode:
            sched = [[(0, 2)]] + [[(0, 1)]] * (n - 2)
        else:
            sched = [[(0, n - 19)], [(0, 19)]]
        got = run_schedule(eng, [toks], sched)[0]
        check(got, want, dtype, f"key {target}")
        for i in range(target + 1, n):
            seen = i - target < window or target < keep
            assert (_moved(got[i].cpu(), without[i]) > 0.2) == seen, (i, target)


def case_far_key(kind, device, dtype, decode, dim=20):
    """One key hundreds of positions back that the last queries point at:
    the first one, one at each side of a page border; unbounded attention,
    and the latent one."""
    cfg, W = pointing(kind, dim=dim, vdim=128 if dim == 128 and
                      kind == "attention" else 8)
    n = 300
    plain = logits_of(cfg, W, [8 + 0] * n)
    for target in (0, 63, 64):
        toks = [8 + 0] * n
        toks[target] = 8 + 1
        want = logits_of(cfg, W, toks)
        assert _moved(want[-1], plain[-1]) > 0.3
        eng = make_engine(cfg, W, device, dtype, block_size=16, max_len=320)
        sched = ([[(0, n - 6)]] + [[(0, 1)]] * 6 if decode
                 else [[(0, 130)], [(0, 170)]])
        got = run_schedule(eng, [toks], sched)[0]
        check(got, want, dtype, f"key {target}")


def case_sink(kind, device, dtype, dim=20):
    """Scores far below the sink (it takes nearly all weight and the output
    nearly vanishes), far above it (it must not matter), and near it; counted
    once whatever the number of keys, passes and cuts."""
    for strength, sink in ((-30.0, 0.0), (0.0, 9.0), (0.0, 0.5), (30.0, 2.0),
                           (0.0, -20.0), (-80.0, -60.0)):
        cfg, W = pointing(kind, strength, dim=dim,
                          vdim=128 if dim == 128 and kind == "attention"
                          else 8)
        W["l0.mix.sink"] = _b(torch.tensor([sink, sink - 1.0]))
        toks = [8 + 1] * 40
        want = logits_of(cfg, W, toks)
        off = dict(W)
        off["l0.mix.sink"] = torch.full((2,), -300.0)
        shows = _moved(want[-1], logits_of(cfg, off, toks)[-1])
        assert (shows > 0.01) == (strength < 0 or -20.0 < sink < 30.0 and
                                  strength == 0.0), (strength, shows)
        eng = make_engine(cfg, W, device, dtype, block_size=16)
        for cuts in ([37, 1, 1, 1], [2, 18, 20], [1] * 40):
            got = run_schedule(eng, [toks], [[(0, k)] for k in cuts])[0]
            check(got, want, dtype, f"{kind} {strength} {sink} {cuts[:3]}")


def faults():
    """Changes of the plain model, one per mechanism: (configuration name,
    what is changed, change(cfg, weights))."""
    def mask(key, by):
        def f(cfg, W):
            for L in cfg["layers"]:
                if "mask" in L["mixer"]:
                    L["mixer"]["mask"][key] += by
        return f

    def rot(kind, **kw):
        def f(cfg, W):
            for L in cfg["layers"]:
                if L["type"] == kind:
                    L["mixer"]["rot"].update(kw)
        return f

    def scal(kind, **kw):
        def f(cfg, W):
            for L in cfg["layers"]:
                if L["type"] == kind:
                    L["mixer"]["rot"]["scaling"].update(kw)
        return f

    def router(**kw):
        def f(cfg, W):
            for L in cfg["layers"]:
                if L["mlp"] and L["mlp"]["kind"] == "moe":
                    r = L["mlp"]["router"]
                    if "groups" in r:
                        r["groups"].update(kw)
        return f

    def zero(end):
        def f(cfg, W):
            for k in W:
                if k.endswith(end):
                    W[k] = torch.zeros_like(W[k])
        return f
    A, Z = "attention", "latent_attention"
    return [
        ("window + 1", mask("size", 1)), ("window - 1", mask("size", -1)),
        ("keep + 1", mask("keep_first", 1)),
        ("keep - 1", mask("keep_first", -1)),
        ("no banded scaling", rot(A, scaling=None)),
        ("no yarn", rot(Z, scaling=None)),
        ("band limit low", scal(A, low=0.5)),
        ("band limit high", scal(A, high=6.0)),
        ("ramp start", scal(Z, fast=1.2)),
        ("ramp end", scal(Z, slow=0.1)),
        ("fewer groups", router(keep=1)),
        ("no correction", zero(".correction")),
        ("sinks at 0", zero(".sink")),
        ("no embedding norm weight", zero("embed.norm")),
    ]


def case_faults_show():
    """Every such change moves the plain model's logits by far more than the
    tolerance of the exact mode: the random weights hide none of them."""
    toks = tokens(CONFIGS["hybrid"](), 40, 5)
    cfg = CONFIGS["hybrid"]()
    base = logits_of(cfg, weights(cfg, 5), toks)
    for name, change in faults():
        c = copy.deepcopy(CONFIGS["hybrid"]())
        W = weights(c, 5)
        if name == "fewer groups":
            for L in c["layers"]:
                if L["mlp"] and L["mlp"]["kind"] == "moe":
                    L["mlp"]["router"]["top"] = 2
            base2 = logits_of(c, W, toks)
        else:
            base2 = base
        change(c, W)
        e = row_errors(logits_of(c, W, toks), base2)
        assert float(e.max()) > 50 * tol("fp32"), \
            f"{name}: {float(e.max()):.3g}"


def case_rotation_tables():
    """Angle tables of every scaling against the plain formulas."""
    for dims, base, scaling in (
            (24, 500.0, None), (2, 10000.0, banded()), (64, 5e5, banded(
                8.0, 1.0, 4.0, 8192)), (16, 20.0, banded(2.0, 1.0, 1.0, 50)),
            (10, 300.0, yarn()), (64, 10000.0, yarn(4.0, 4096, 32.0, 1.0)),
            (4, 1e6, yarn(40.0, 16, 1.5, 1.2)), (8, 2.0, yarn(1.0))):
        f, amp = oracle.rotation({"dims": dims, "base": base,
                                  "scaling": scaling})
        n = 50
        ang = torch.arange(n, dtype=torch.float64)[:, None] * torch.tensor(
            f, dtype=torch.float64)[None]
        want = torch.cat([ang.cos(), ang.sin()], 1) * amp
        _close(angle_table(n, dims, base, scaling), want, "fp32",
               f"{dims} {base} {scaling}")


def case_feed_forwards(device, dtype):
    """Both feed-forwards alone against the plain model; routed experts with
    every kind of grouping, rows in both forms of the expert pass."""
    from kukeon_amd.models.senavik import FEED_FORWARDS
    for f, Wd, T in ((dense(9), 22, 5), (dense(72), 40, 70),
                     (moe(6, 2, 10, (3, 2)), 24, 5),
                     (moe(8, 3, 24, (2, 1)), 40, 70),
                     (moe(4, 4, 8, (4, 4)), 24, 66), (moe(5, 1, 9), 22, 3),
                     (moe(12, 4, 72, (6, 3)), 136, 40),
                     (moe(2, 2, 64, (1, 1)), 256, 63)):
        cfg = config([layer(attn(), f)], width=Wd)
        W = weights(cfg, 30 + T)
        t64 = {k: v.double() for k, v in W.items()}
        g = torch.Generator().manual_seed(T)
        h = torch.randn(T, Wd, generator=g).to(torch.bfloat16)
        want = oracle.dense(h.double(), t64, "l0.mlp.") \
            if f["kind"] == "dense" else oracle.moe(h.double(), t64,
                                                    "l0.mlp.", f)
        fc = SenavikConfig.from_json(cfg).layers[0].mlp
        mod = FEED_FORWARDS[fc.kind](fc, Wd, W, "l0.mlp.", device,
                                     _act(dtype))

        class Meta:
            host_ids = list(range(T))
        for meta in (Meta(), None):
            got = mod(h.to(device=device, dtype=_act(dtype)), None, meta)
            check(got, want, dtype, f"{f}")


# ------------------------------------------------------- single operations
def case_op_norms(device, dtype):
    """The stack's start (embedding row, norm, first layer's norm) and the
    residual sum with the next norm, weights stored around zero."""
    from kukeon_amd import ops
    g = torch.Generator().manual_seed(5)
    act = _act(dtype)
    for Wd in (16, 26, 40, 2048, 4096, 8192, 8200):
        T, V, eps = 5, 11, 1e-3
        table = torch.randn(V, Wd, generator=g).to(act) * 0.2
        w, w2 = (torch.randn(Wd, generator=g) * 0.3 for _ in range(2))
        ids = torch.tensor([3, 10, 0, 3, 7], dtype=torch.int32)
        cfg = {"norm": {"eps": eps}}
        want = oracle.embed(ids.tolist(), {"embed": table.double(),
                                           "embed.norm": w.double()}, cfg)
        x = torch.full((T, Wd), 9.0, device=device)
        h = torch.full((T, Wd), 9.0, dtype=act, device=device)
        d = lambda t: t.to(device)
        ops.embed_rmsnorm(x, h, d(ids), d(table), d(w), d(w2), 1.0, eps)
        _close(x, want, "fp32", f"{Wd}: stream")
        _close(h, oracle.offset_norm(want, w2.double(), cfg), dtype,
               f"{Wd}: first input")
        y = torch.randn(T, Wd, generator=g).to(act)
        ops.residual_add_rmsnorm(x, d(y), None, d(w2), 1.0, eps, h)
        want = want + y.double()
        _close(x, want, "fp32", f"{Wd}: sum")
        _close(h, oracle.offset_norm(want, w2.double(), cfg), dtype,
               f"{Wd}: next input")


def case_op_rotary(device, dtype):
    """Partial rotation and the page writes, three sequences of which one is
    inactive, sizes on and off the vector path."""
    from kukeon_amd import ops
    g = torch.Generator().manual_seed(12)
    act = _act(dtype)
    for H, G, d, dv, dims, BS in ((3, 1, 7, 5, 4, 4), (4, 2, 24, 16, 20, 16),
                                  (2, 2, 128, 128, 128, 16),
                                  (6, 3, 16, 40, 0, 4), (5, 5, 8, 8, 2, 4)):
        cuts, start = [7, 2, 5], [3, -1, 0]
        T = sum(cuts)
        qc, kc_, vc_ = G * (d + dv) + 8, 0, G * d
        proj = torch.randn(T, qc + H * d + 8, generator=g).to(act)
        pos, row_seq, _, _ = _maps(cuts, start, device, [0, 1, 2])
        bt = torch.tensor([[5, 1, 3], [0, 0, 0], [2, 4, 6]],
                          dtype=torch.int32, device=device)
        rot = {"dims": dims, "base": 12.0}
        cs = angle_table(20, dims, 12.0).to(device) if dims else \
            torch.zeros(20, 0, device=device)
        kc = torch.full((8, G, BS, d), 7.0, dtype=act, device=device)
        vc = torch.full((8, G, BS, dv), 7.0, dtype=act, device=device)
        qo = torch.full((T, H * d), 7.0, dtype=act, device=device)
        ops.rotary_append(qo, kc, vc, proj.to(device), qc, kc_, vc_, cs, pos,
                          row_seq, bt)
        # the kernel turns neighbours; the plain model halves
        half = list(range(0, dims, 2)) + list(range(1, dims, 2)) + \
            list(range(dims, d))
        back = torch.tensor(half).argsort()
        want_k = torch.full((8, G, BS, d), 7.0, dtype=torch.float64)
        want_v = torch.full((8, G, BS, dv), 7.0, dtype=torch.float64)
        for r in range(T):
            p = int(pos[r])
            if p < 0:
                continue

            def turned(x, n):
                z = torch.zeros(p + 1, n, d, dtype=torch.float64)
                z[p] = x.double().view(n, d)[:, half]
                return oracle.rotate(z, rot)[p][:, back]
            _close(qo[r], turned(proj[r, qc: qc + H * d], H).reshape(-1),
                   dtype, "queries")
            b = int(bt[int(row_seq[r]), p // BS])
            want_k[b, :, p % BS] = turned(proj[r, : G * d], G)
            want_v[b, :, p % BS] = proj[r, vc_: vc_ + G * dv].double().view(
                G, dv)
        _close(kc, want_k, dtype, "key pages")
        assert torch.equal(vc.cpu().double(), want_v)


def case_op_attention(device, dtype, d=8, dv=8, BS=4, n=90, start=0):
    """Windowed attention with kept tokens, sinks and values of their own
    against dense scores, with and without each. One query and key pair is
    scaled up so that its score stands out, at the window's edge, at the last
    kept token and one place outside both."""
    from kukeon_amd import ops
    g = torch.Generator().manual_seed(11 + d)
    H, G = 6, 2
    act = _act(dtype)
    nb = -(-n // BS)
    perm = torch.randperm(nb, generator=g)
    k = torch.randn(n, G, d, generator=g).to(act)
    v = torch.randn(n, G, dv, generator=g).to(act)
    q = torch.randn(n - start, H * d, generator=g).to(act)
    window, keep = 33, 5
    for row, key in ((n - 1, n - window), (n - 2, n - 2 - window),
                     (n - 3, keep - 1), (n - 4, keep)):
        q[row - start] = (k[key].repeat_interleave(H // G, 0).reshape(-1) *
                          1.5).to(act)
    sinks = torch.randn(H, generator=g) * 2 + 1
    kc = torch.full((nb, G, BS, d), 300.0, dtype=act)
    vc = torch.full((nb, G, BS, dv), 300.0, dtype=act)
    for j in range(n):
        kc[perm[j // BS], :, j % BS] = k[j]
        vc[perm[j // BS], :, j % BS] = v[j]
    pos, row_seq, _, _ = _maps([n - start], [start], device, [0])
    bt = perm.to(torch.int32)[None].to(device).contiguous()
    dd = lambda t: t.to(device)
    scale = 1.5 * d ** -0.5
    for w, kp, sk in ((window, keep, True), (window, 0, True),
                      (window, keep, False), (0, 0, True), (0, 7, False),
                      (1, 2, True), (n + 5, keep, True), (20, 70, True)):
        want = torch.zeros(n - start, H, dv, dtype=torch.float64)
        for i in range(start, n):
            js = oracle.visible(i, {"size": w, "keep_first": kp})
            for h in range(H):
                s = k[js, h // (H // G)].double() @ \
                    q[i - start].double().view(H, d)[h] * scale
                want[i - start, h] = oracle.sink_weights(
                    s, sinks[h].double() if sk else None) @ \
                    v[js, h // (H // G)].double()
        want = want.view(n - start, H * dv)
        out = torch.full((n - start, H * dv), 9.0, dtype=act, device=device)
        ops.masked_attention(out, dd(q), dd(kc), dd(vc), None, None, None,
                             pos, row_seq, bt, H, scale, window=w,
                             sinks=dd(sinks) if sk else None, keep=kp)
        _close(out, want, dtype, f"rows {w} {kp} {sk}")
        if not ops.masked_tiles_supported(dd(q), d, BS, dv):
            continue
        i32 = lambda t: torch.tensor(t, dtype=torch.int32, device=device)
        qb = list(range(0, n - start, 32))
        out = torch.full((n - start, H * dv), 9.0, dtype=act, device=device)
        ops.masked_attention_tiles(
            out, dd(q), dd(kc), dd(vc), None, None,
            dd(sinks) if sk else None, bt, i32([n]), i32([[start, 0]]),
            i32([0] * len(qb)), i32(qb), scale, window=w, keep=kp)
        _close(out, want, dtype, f"tiles {w} {kp} {sk}")


def case_op_latent(device, dtype, H=5, R=24, dr=6, n=70, BS=4, rows=None):
    """Latent attention with a sink per head, every row and single rows (the
    keys of which the kernels share out), beside an inactive row."""
    from kukeon_amd import ops
    g = torch.Generator().manual_seed(R + n)
    act = _act(dtype)
    dn = 8
    qa = (torch.randn(H, n, R, generator=g) * 0.4).to(act)
    q = torch.randn(n, H * (dn + dr), generator=g).to(act)
    lat = torch.randn(n, R, generator=g).to(act)
    kr = torch.randn(n, dr, generator=g).to(act)
    sinks = torch.randn(H, generator=g) * 2 + 2
    nb = -(-n // BS)
    perm = torch.randperm(nb, generator=g)
    cache = torch.full((nb, 1, BS, R + dr), 300.0, dtype=act)
    for j in range(n):
        cache[perm[j // BS], 0, j % BS] = torch.cat([lat[j], kr[j]])
    scale = 0.3
    ids = rows if rows is not None else list(range(n))
    want = torch.zeros(H, len(ids), R, dtype=torch.float64)
    for a, i in enumerate(ids):
        for h in range(H):
            s = lat[: i + 1].double() @ qa[h, i].double() + \
                kr[: i + 1].double() @ \
                q[i].double().view(H, dn + dr)[h, dn:]
            want[h, a] = oracle.sink_weights(
                s * scale, sinks[h].double()) @ lat[: i + 1].double()
    # angles of zero: the rotated parts stay as they are
    cs = torch.cat([torch.ones(n, dr // 2), torch.zeros(n, dr // 2)],
                   1).to(device).contiguous()
    bt = perm.to(torch.int32)[None].to(device).contiguous()

    def run(at):
        m = len(at)
        out = torch.full((H, m, R), 9.0, dtype=act, device=device)
        src = [max(i, 0) for i in at]
        ops.latent_attention(
            out, qa[:, src].contiguous().to(device), q[src].to(device),
            cache.to(device), cs,
            torch.tensor(at, dtype=torch.int32, device=device),
            torch.zeros(m, dtype=torch.int32, device=device), bt, H, dn, dr,
            0, scale, sinks.to(device))
        return out
    _close(run(ids), want, dtype, f"rows {R} {dr}")
    few = [ids[-1], -1, ids[0], ids[len(ids) // 2]]
    out = run(few)
    assert float(out[:, 1].abs().max()) == 0.0
    for a, i in enumerate(few):
        if i >= 0:
            _close(out[:, a], want[:, ids.index(i)], dtype, f"row {i} of few")


def case_op_heads(device, dtype):
    """Heads brought together without a gate."""
    from kukeon_amd import ops
    g = torch.Generator().manual_seed(4)
    for H, T, dv in ((3, 5, 7), (4, 9, 16)):
        o = torch.randn(H, T, dv, generator=g).to(_act(dtype)).to(device)
        out = torch.full((T, H * dv), 9.0, dtype=_act(dtype), device=device)
        ops.head_gate(out, o, None)
        assert torch.equal(out.cpu(), o.cpu().permute(1, 0, 2).reshape(
            T, H * dv))


def case_op_router(device):
    """Corrected choice in groups against the plain one: every grouping,
    negative choice scores, ties, experts over several lanes, rows wider than
    needed, a NaN."""
    from kukeon_amd import ops
    g = torch.Generator().manual_seed(8)
    for E, top, groups in ((6, 2, (3, 2)), (8, 3, None), (4, 4, (4, 4)),
                           (17, 2, None), (12, 5, (4, 2)), (160, 8, (8, 3)),
                           (5, 1, (5, 1)), (130, 70, (65, 40)),
                           (9, 3, (3, 1)), (1, 1, None)):
        T = 40
        z = torch.randn(T, E, generator=g) * 2
        c = torch.randn(E, generator=g) * 0.5 - 0.8
        z[3] = 0.25
        pick, w = oracle.route(
            z.double(), {"x.router": torch.eye(E, dtype=torch.float64),
                         "x.correction": c.double()}, "x.",
            {"top": top, "groups": groups and {"count": groups[0],
                                               "keep": groups[1]}})
        wide = torch.zeros(T, E + 3)
        wide[:, :E] = z
        idx = torch.full((T, top + 1), -5, dtype=torch.int32, device=device)
        wts = torch.zeros(T, top + 1, device=device)
        n, keep = groups or (0, 0)
        ops.router_corrected(idx, wts, wide.to(device)[:, :E], c.to(device),
                             top, n, keep, 2, 1.0, True)
        assert torch.equal(idx[:, :top].cpu().long(), pick), (E, top, groups)
        assert int(idx[:, top].max()) == -5
        _close(wts[:, :top], w, "fp32", f"weights {E}")
    # equal scores: the lowest indices of the lowest groups
    idx = torch.zeros(1, 3, dtype=torch.int32, device=device)
    wts = torch.zeros(1, 3, device=device)
    ops.router_corrected(idx, wts, torch.zeros(1, 8, device=device), None, 3,
                         4, 2, 1, 2.0, False)
    assert idx[0].tolist() == [0, 1, 2]
    _close(wts, torch.full((1, 3), 1.0), "fp32", "plain scores times scale")
    # a group's best alone or its two best together
    z = torch.logit(torch.tensor([[0.9, 0.1, 0.6, 0.55, 0.2, 0.3]])).to(device)
    for best, want in ((1, [0, 1]), (2, [2, 3])):
        idx = torch.zeros(1, 2, dtype=torch.int32, device=device)
        ops.router_corrected(idx, torch.zeros(1, 2, device=device), z, None,
                             2, 3, 1, best, 1.0, True)
        assert idx[0].tolist() == want
    if torch.device(device).type != "cpu":
        z = torch.randn(4, 6, generator=g).to(device)
        z[1] = float("nan")
        idx = torch.zeros(4, 2, dtype=torch.int32, device=device)
        wts = torch.zeros(4, 2, device=device)
        ops.router_corrected(idx, wts, z, None, 2, 3, 2, 2, 1.0, True)
        assert 0 <= int(idx.min()) and int(idx.max()) < 6
        assert bool(torch.isfinite(wts).all())


# ------------------------------------------------- folders, programs, servers
def case_registry(tmp_path, device, dtype):
    """A checkpoint folder is found by its architecture name and read."""
    from dumovik_cases import write_checkpoint
    from kukeon_amd.models.registry import load_checkpoint
    cfg = CONFIGS["only_latent"]()
    W = weights(cfg, 11)
    write_checkpoint(tmp_path, cfg, W)
    mcfg, model = load_checkpoint(str(tmp_path), device=device, dtype=dtype)
    assert mcfg.family == "senavik" and len(model.layers) == 2
    eng = LLMEngine(model, mcfg, EngineConfig(
        block_size=4, max_model_len=64, max_sessions=2, num_kv_blocks=16,
        use_graphs=False), device=device)
    toks = tokens(cfg, 13, 11)
    got = run_schedule(eng, [toks], [[(0, 6)], [(0, 7)]])[0]
    check(got, logits_of(cfg, W, toks, got), dtype, "from a folder")


def case_trace_runner(tmp_path, device, dtype):
    """The trace runner as a program: a checkpoint folder, steps on standard
    input, logits files and `done` lines back. Three requests through a pool
    sized for two, portions beside single tokens, a request left out of a
    step."""
    import json
    import os
    import subprocess
    import sys
    import numpy as np
    from dumovik_cases import write_checkpoint
    cfg = CONFIGS["hybrid"]()
    W = weights(cfg, 14)
    model_dir, out_dir = tmp_path / "model", tmp_path / "out"
    model_dir.mkdir()
    write_checkpoint(model_dir, cfg, W)
    prompts = {"a": tokens(cfg, 70, 90), "b": tokens(cfg, 40, 91),
               "c": tokens(cfg, 33, 92)}
    want = {k: logits_of(cfg, W, p) for k, p in prompts.items()}
    steps = [[("a", 30), ("b", 1)], [("a", 1), ("b", 38)], [("a", 39)],
             [("b", 1), ("c", 2)], [("c", 30)], [("c", 1)]]
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    cmd = [sys.executable, os.path.join(root, "bin", "trace_run"), "--model",
           str(model_dir), "--dtype",
           "float32" if dtype == "fp32" else "bfloat16", "--out",
           str(out_dir), "--max-tokens", "128", "--slots", "2", "--device",
           device]
    p = subprocess.Popen(cmd, stdin=subprocess.PIPE, stdout=subprocess.PIPE,
                         text=True, cwd=root)
    at = {k: 0 for k in prompts}
    rows, files = [], []
    try:
        for n, step in enumerate(steps):
            entries, end = [], []
            for k, cnt in step:
                toks = prompts[k][at[k]: at[k] + cnt]
                entries.append({"id": k, "tokens": toks,
                                "want": [0, cnt - 1] if cnt > 1 else [0]})
                at[k] += cnt
                if at[k] == len(prompts[k]):
                    end.append(k)
            p.stdin.write(json.dumps({"step": n, "entries": entries,
                                      "end": end}) + "\n")
            p.stdin.flush()
            line = p.stdout.readline()
            while line and line.strip() != "done %d" % n:
                line = p.stdout.readline()
            assert line, "the runner ended early"
            files.append(torch.from_numpy(np.fromfile(
                out_dir / ("%d.f32" % n), dtype="<f4").reshape(
                -1, cfg["vocab"])))
            rows += [want[k][at[k] - cnt + w] for k, cnt in step
                     for w in ([0, cnt - 1] if cnt > 1 else [0])]
        p.stdin.close()
        assert p.wait(timeout=60) == 0
    finally:
        if p.poll() is None:
            p.kill()
    got = torch.cat(files)
    assert got.shape[0] == len(rows)
    if dtype == "fp32":
        check(got, torch.stack(rows), dtype, "runner")
    else:       # a router's close call may fall either way
        e = row_errors(got, torch.stack(rows))
        assert float(e.median()) <= 0.4 * tol(dtype)


def case_modelhub(device):
    """The serving daemon's model server with this family: sessions over the
    unix socket, two turns on one session, greedy tokens as the plain model
    gives them."""
    import uuid
    from kukeon_amd.serve.server import ModelhubClient, ModelhubServer
    cfg = CONFIGS["hybrid"]()
    W = weights(cfg, 16)
    mcfg = SenavikConfig.from_json(cfg)
    model = SenavikModel(mcfg, device=device, dtype="fp32", tensors=W,
                         max_position=128)
    ecfg = EngineConfig(block_size=4, max_model_len=128, max_sessions=4,
                        num_kv_blocks=64, use_graphs=False)
    sock = f"/tmp/mh-{uuid.uuid4().hex[:10]}.sock"
    hub = ModelhubServer(model, mcfg, ecfg, sock, device=device)
    hub.start()
    try:
        c = ModelhubClient(sock, timeout=120)
        p1, p2 = tokens(cfg, 6, 70), tokens(cfg, 3, 71)
        r1 = c.generate("s", p1, max_new_tokens=4, temperature=0.0)
        assert len(r1["tokens"]) == 4
        assert_greedy(cfg, W, p1, r1["tokens"], "first turn")
        r2 = c.generate("s", p2, max_new_tokens=3, temperature=0.0)
        assert len(r2["tokens"]) == 3
        assert_greedy(cfg, W, p1 + r1["tokens"] + p2, r2["tokens"],
                      "second turn")
        rb = c.generate("t", p2, max_new_tokens=2, temperature=0.0)
        assert_greedy(cfg, W, p2, rb["tokens"], "other session")
        assert c.call("stats")["sessions"] == 2
        c.close()
    finally:
        hub.stop()


def case_real_sizes(device, say=lambda s: None):
    """A stack at the layer sizes of a served model (heads of 128, pages of
    16, a latent of 512, rows of thousands of entries): the bf16 serving
    kernels against the exact fp32 kernels, prompts on the packed path and
    decoding under hipGraphs."""
    from kukeon_amd.models.senavik import random_tensors, senavik_bench
    mcfg = senavik_bench(width=2048, layers=4, heads=16, kv_heads=4, ff=4096,
                         vocab=512, window=96, experts=16,
                         name="senavik-sizes")
    W = random_tensors(mcfg, 5)
    g = torch.Generator().manual_seed(9)
    prompts = [torch.randint(0, 512, (n,), generator=g).tolist()
               for n in (150, 70, 129)]
    outs = {}
    for dtype in ("fp32", "bf16"):
        say(f"model {dtype}")
        model = SenavikModel(mcfg, device=device, dtype=dtype, tensors=W)
        eng = LLMEngine(model, mcfg, EngineConfig(
            block_size=16, max_model_len=512, max_sessions=4,
            num_kv_blocks=64, use_graphs=False), device=device)
        say("prompts")
        kvs = [SequenceKV(16) for _ in prompts]
        lg = [eng.forward_tokens([(kv, p[:-6]) for kv, p in
                                  zip(kvs, prompts)])]
        say("single tokens")
        for k in range(6, 0, -1):
            lg.append(eng.forward_tokens([(kv, [p[-k]]) for kv, p in
                                          zip(kvs, prompts)]))
        outs[dtype] = torch.cat(lg).float().cpu()
        assert bool(torch.isfinite(outs[dtype]).all())
        for kv in kvs:
            eng.free_sequence(kv)
        if dtype == "bf16":
            say("generation under graphs")
            eng.ecfg.use_graphs = True
            eng.ecfg.graph_buckets = (4,)
            eng.ecfg.decode_microbatch = 8
            sp = SamplingParams(temperature=0.7, top_k=50, top_p=0.9,
                                max_new_tokens=17)
            kvs = [SequenceKV(16) for _ in prompts]
            rids = [eng.add_request(kv, p, sp) for kv, p in
                    zip(kvs, prompts)]
            n = 0
            while eng.has_work():
                for o in eng.step():
                    n += len(o.new_tokens)
                    assert all(0 <= t < 512 for t in o.new_tokens)
            assert n == 17 * len(rids)
        del eng, model
    e = row_errors(outs["bf16"], outs["fp32"])
    over = int((e > 0.15).sum())
    assert over <= max(1, e.numel() // 4), f"{over} rows off, worst " \
        f"{float(e.max()):.3g}"
