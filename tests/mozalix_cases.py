"""The Mozalix test cases, parametrised by device and dtype.  Each case builds its own small configuration, writes a
checkpoint from the plain oracle's random weights (``mozalix_oracle``), replays step schedules through the engine
(``rodelix_common.Rig``: the engine's runner, block manager, cache, state slots and kernels) and compares every position's
logits with the oracle.  The same cases run on the CPU path (``test_mozalix.py``) and on the GPU kernels
(``test_mozalix_gpu.py``)."""
from __future__ import annotations

import copy
import json
import os

import torch

import mozalix_oracle as oracle
from rodelix_common import Rig, TOL, alone, chunks, rel_err, tokens

DENSE = {"kind": "dense", "ff": 92, "limit": 1.6}


def chunk(heads=6, kv_heads=2, dim=20, vdim=12, size=37, dims=8, base=2000.0, scale=0.3, mlp=None):
    return {"type": "attention", "mlp": copy.deepcopy(mlp),
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "mask": {"size": size},
                      "rot": {"base": base, "dims": dims}}}


def diff(heads=4, kv_heads=2, dim=12, vdim=20, size=19, dims=12, base=700.0, scale=0.35, lam=0.3, mlp=None):
    return {"type": "attention_2", "mlp": copy.deepcopy(mlp),
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "diff": lam, "mask": {"size": size},
                      "rot": {"base": base, "dims": dims}}}


def capped(heads=3, kv_heads=1, dim=16, vdim=28, size=11, keep=2, cap=3.0, scale=0.4):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "softcap": cap, "mask": {"size": size, "keep_first": keep}}


def delta(heads=6, kv_heads=2, dim=12, vdim=20, conv=3):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}


def pair(left=None, right=None, scales=(0.5, 1.2), mlp=None):
    return {"type": "parallel", "mlp": copy.deepcopy(mlp),
            "mixer": {"left": left or capped(), "right": right or delta(), "left_scale": scales[0], "right_scale": scales[1]}}


def again(i):
    return {"again": i}


def make_cfg(layers, width=72, vocab=151, scale=0.8, eps=1e-5):
    out = []
    for l in layers:
        out.append(dict(copy.deepcopy(out[l["again"]]), weights_of=l["again"]) if "again" in l else copy.deepcopy(l))
    return {"architecture": "Mozalix", "vocab": vocab, "width": width, "embedding": {"scale": scale}, "norm": {"eps": eps}, "layers": out}


# every mixer, with and without a feed-forward, sizes of their own, three layers on others' weights (one of them through another)
FULL = make_cfg([diff(mlp=DENSE), chunk(mlp=DENSE), pair(mlp=DENSE), again(1),
                 pair(capped(4, 2, 12, 16, 40, 0, 8.0), delta(4, 4, 16, 8, 5), (0.5, 1.1)), again(2), again(0), again(3)])


def write_checkpoint(path, cfg, seed=0, bf16=False, edit=None, ranks=(6, 10)):
    """config.json + model.safetensors; returns the weights as stored (fp32 values) for the oracle."""
    from safetensors.torch import save_file
    os.makedirs(path, exist_ok=True)
    W = oracle.random_weights(cfg, seed, ranks)
    if edit:
        edit(W)
    if bf16:
        W = {k: v.to(torch.bfloat16) for k, v in W.items()}
    with open(os.path.join(path, "config.json"), "w") as fh:
        json.dump(cfg, fh)
    save_file({k: v.contiguous() for k, v in W.items()}, os.path.join(path, "model.safetensors"))
    return {k: v.float() for k, v in W.items()}


def expect(cfg, W, toks, faults=()):
    return oracle.forward(resolved(cfg), W, toks, faults)[0].numpy()


def resolved(cfg):
    """The oracle takes the tensors of the layer ``weights_of`` names: follow chains to the layer that owns them."""
    cfg = copy.deepcopy(cfg)
    for L in cfg["layers"]:
        while L.get("weights_of") is not None and cfg["layers"][L["weights_of"]].get("weights_of") is not None:
            L["weights_of"] = cfg["layers"][L["weights_of"]]["weights_of"]
    return cfg


def _setup(tmp, cfg, dtype, device, seed=0, edit=None, ranks=(6, 10), **rig):
    W = write_checkpoint(tmp, cfg, seed, bf16=dtype == "bfloat16", edit=edit, ranks=ranks)
    return W, Rig(tmp, dtype, device, **rig)


def _check(got, want, dtype, what="", single=False):
    """Every row within the tolerance.  In bf16 the small heads of these stacks leave single rows with three times the rounding of the
    others (a difference of two maps, a recurrence's output near zero, divided by its root mean square): there the rows' median
    has to be well inside, unless the stack is a ``single`` layer."""
    e = rel_err(got, want)
    loose = 2.5 if dtype == "bfloat16" and not single else 1.0
    assert e < loose * TOL[dtype], f"{what}: relative error {e:.3e} over {loose * TOL[dtype]:.1e}"
    if loose > 1.0:
        mid = sorted(rel_err(got[[i]], want[[i]]) for i in range(len(want)))[len(want) // 2]
        assert mid < 0.6 * TOL[dtype], f"{what}: median relative error {mid:.3e}"


# ---------------------------------------------------------------- each mechanism alone
def _silence(*ends):
    def edit(Wt):
        for k in Wt:
            if k.endswith(ends):
                Wt[k] = Wt[k] * 0.0
    return edit


MECHANISMS = {
    "chunked attention": (make_cfg([chunk(), chunk(heads=3, kv_heads=3, dim=16, vdim=24, size=8, dims=16)]), None),
    "differential attention": (make_cfg([diff(), diff(heads=3, kv_heads=1, dim=20, vdim=28, size=33, dims=4)]), None),
    "capped window attention": (make_cfg([pair(), pair(capped(4, 4, 20, 12, 9, 2, 1.5))]), _silence("right.o")),
    "delta rule": (make_cfg([pair(), pair(right=delta(2, 1, 24, 16, 1))]), _silence("left.o")),
    "scaled pair": (make_cfg([pair(), pair(scales=(1.2, 0.3))]), None),
    "feed-forward": (make_cfg([chunk(mlp=DENSE), diff(mlp=DENSE), pair(mlp=DENSE)]), _silence("mix.o", "left.o", "right.o")),
    "shared weights": (make_cfg([diff(mlp=DENSE), again(0), pair(), again(2), again(1)]), None),
}


def case_mechanism(tmp, device, dtype, kind):
    cfg, edit = MECHANISMS[kind]
    W, rig = _setup(tmp, cfg, dtype, device, seed=3, edit=edit)
    toks = tokens(150, cfg["vocab"], 1)
    want = expect(cfg, W, toks)
    _check(rig.run({"a": toks}, alone("a", len(toks), [len(toks)]))["a"], want, dtype, f"{kind} whole prompt")
    _check(rig.run({"b": toks}, alone("b", len(toks), [31, 2, 1, 40, 1, 1, 7]))["b"], want, dtype, f"{kind} in portions")


# ---------------------------------------------------------------- getting a mechanism wrong must show
FAULTS = ("embed_scale", "norm_offset", "pre_norm", "shared", "qk_norm", "qk_weight", "late_norm", "rotation", "chunk", "chunk_size", "sink",
          "window", "narrow", "keep", "keep_more", "softcap", "one_map", "lambda", "map_norm", "map_scale", "map_heads", "scales", "conv",
          "conv_act", "unit", "q_scale", "beta", "decay", "head_decay", "erase", "late_read", "dt_bias", "out_norm", "gate", "limit", "up_offset",
          "gate_slope", "ff_bias")


def _telling(Wt):
    """Weights under which every single mistake moves the logits: peaked scores, heavy sinks, decays that differ over the channels."""
    for k in list(Wt):
        if k.endswith("sink"):
            Wt[k] = Wt[k] + 2.5
        if k.endswith("right.a2"):
            Wt[k] = Wt[k] * 2.5
        if k.endswith(("right.q", "right.k")):
            Wt[k] = Wt[k] * 0.05                                # unit vectors from short ones: their length matters
        if k.endswith("right.v"):
            Wt[k] = Wt[k] * 0.02                                # outputs near the norm's epsilon
        if k.endswith(("q.norm", "k.norm")):
            Wt[k] = Wt[k] + 0.5
        if k.endswith("mix.o") and k[:-1] + "lq1" in Wt:
            Wt[k] = Wt[k] * 0.004                               # the norm behind the maps sees its epsilon: their scale matters


def case_each_piece_matters(tmp, device, dtype):
    W, rig = _setup(tmp, FULL, dtype, device, seed=4, edit=_telling)
    toks = tokens(70, FULL["vocab"], 2)
    want = expect(FULL, W, toks)
    for fault in FAULTS:
        # the oracle itself must tell these faults, or the comparison below shows nothing
        off = rel_err(expect(FULL, W, toks, (fault,)), want)
        assert off > 3 * TOL[dtype], f"{fault}: {off:.2e}"
    _check(rig.run({"p": toks}, alone("p", 70, [70]))["p"], want, dtype, "prompt")
    _check(rig.run({"d": toks}, alone("d", 70, [20, 2, 3] + [1] * 45))["d"], want, dtype, "portions and decoding")


# ---------------------------------------------------------------- prefill against token-by-token, portions down to two
def case_prefill_decode_portions(tmp, device, dtype):
    W, rig = _setup(tmp, FULL, dtype, device, seed=5)
    toks = tokens(135, FULL["vocab"], 2)
    want = expect(FULL, W, toks)
    for name, sizes in (("whole", [135]), ("one by one", [1]), ("portions", [2, 3, 64, 5, 2, 17]), ("page edges", [32, 32, 1, 31, 4]),
                        ("block edges", [63, 2, 65, 5]), ("sub-block edges", [16, 17, 15, 33]), ("chunk edges", [37, 36, 1, 38]),
                        ("shorter than the convolutions", [2, 1, 2, 2, 1, 1, 3, 88])):
        _check(rig.run({name: toks}, alone(name, len(toks), sizes))[name], want, dtype, name)


# ---------------------------------------------------------------- unequal requests in one batch against each alone
def case_mixed_batch(tmp, device, dtype):
    W, rig = _setup(tmp, FULL, dtype, device, seed=7, max_tokens=512)
    reqs = {"s1": tokens(1, FULL["vocab"], 10), "s23": tokens(23, FULL["vocab"], 11), "m70": tokens(70, FULL["vocab"], 12),
            "l150": tokens(150, FULL["vocab"], 13)}
    want = {i: expect(FULL, W, t) for i, t in reqs.items()}
    plan = {"s1": [1], "s23": [2, 1, 1, 16, 1, 1, 1], "m70": chunks(70, [33, 1, 1, 2, 1]), "l150": chunks(150, [40, 3, 1, 1, 70, 1])}
    sched, k = [], 0
    while any(plan.values()):
        step = [(i, plan[i].pop(0)) for i in ("l150", "s23", "m70", "s1") if plan[i] and (k % 3 != 2 or i != "s23")]
        k += 1
        if step:
            sched.append(step)
    got = rig.run(reqs, sched)
    for i in reqs:
        _check(got[i], want[i], dtype, f"request {i} in mixed batches")


def case_mixed_batch_on_tiles(tmp, device, dtype):
    """Chunks of two sequences beside single tokens of others in one step, with sizes the matrix-core attention kernels take."""
    cfg = other_size_configs()["matrix-core shapes, eight heads on one key head"]
    W, rig = _setup(tmp, cfg, dtype, device, seed=21, max_tokens=640)
    reqs = {"a": tokens(150, cfg["vocab"], 50), "b": tokens(97, cfg["vocab"], 51), "c": tokens(40, cfg["vocab"], 52),
            "d": tokens(3, cfg["vocab"], 53)}
    want = {i: expect(cfg, W, t) for i, t in reqs.items()}
    sched = [[("a", 70), ("c", 33)], [("a", 1), ("b", 64), ("c", 1), ("d", 1)], [("a", 50), ("b", 1), ("c", 1), ("d", 2)],
             [("a", 1), ("b", 32), ("c", 5)], [("a", 28)]]
    got = rig.run(reqs, sched)
    for i in reqs:
        _check(got[i], want[i], dtype, f"request {i} beside the others")


# ---------------------------------------------------------------- pages and state slots freed and used again
def case_reuse(tmp, device, dtype):
    W, rig = _setup(tmp, FULL, dtype, device, seed=9, max_tokens=160, max_seqs=2)      # five pages, two slots
    reqs = {f"r{j}": tokens(n, FULL["vocab"], 20 + j) for j, n in enumerate([70, 45, 64, 33, 80, 5])}
    want = {i: expect(FULL, W, t) for i, t in reqs.items()}
    sched = ([[("r0", 40), ("r1", 45)], [("r0", 30)]] +
             [[("r2", 30), ("r3", 2)], [("r3", 31), ("r2", 1)], [("r2", 33)]] +
             [[("r4", 64)], [("r4", 1), ("r5", 5)], [("r4", 15)]])
    got = rig.run(reqs, sched)
    for i in reqs:
        _check(got[i], want[i], dtype, f"request {i} after reuse")
    # one-token prompts in slots whose last owner left states and convolution inputs behind
    singles = {f"s{j}": tokens(4, FULL["vocab"], 30 + j) for j in range(3)}
    got = rig.run(singles, [[("s0", 1), ("s1", 1)], [("s0", 1), ("s1", 3)], [("s0", 2)], [("s2", 1)], [("s2", 1)], [("s2", 2)]])
    for i in singles:
        _check(got[i], expect(FULL, W, singles[i]), dtype, f"request {i} starting with one token")
    bm = rig.rep.bm
    assert bm.num_free == bm.num_blocks and bm.num_free_state_slots == 2


# ---------------------------------------------------------------- memory of the recurrence
def _remember(Wt):
    for k in list(Wt):
        if k.endswith("A_log"):
            Wt[k] = Wt[k] - 5.0                               # states remember hundreds of tokens
        if k.endswith("dt_bias"):
            Wt[k] = Wt[k] - 2.0


MEMORY = make_cfg([pair(right=delta(dim=32, vdim=24)), pair(right=delta(4, 2, 40, 16))], width=64)


def case_far_token(tmp, device, dtype):
    def edit(Wt):
        _remember(Wt)
        _silence("left.o")(Wt)
    W, rig = _setup(tmp, MEMORY, dtype, device, seed=13, edit=edit)
    toks = tokens(330, MEMORY["vocab"], 4)
    want = expect(MEMORY, W, toks)
    changed = list(toks)
    changed[1] = (toks[1] + 17) % MEMORY["vocab"]             # position 1 must reach the last rows
    assert rel_err(expect(MEMORY, W, changed)[-20:], want[-20:]) > 5 * TOL[dtype]
    _check(rig.run({"p": toks}, alone("p", 330, [300] + [1] * 30))["p"], want, dtype, "far token, prompt then decoding")
    _check(rig.run({"c": toks}, alone("c", 330, [64, 63, 2, 129]))["c"], want, dtype, "far token, portions")


# ---------------------------------------------------------------- one key at an edge
# mask → (layer, its prefix, faults that move an edge, place of the key, tokens that see it, tokens that do not)
SIZE = 45


def _edge(kind, place):
    if kind == "chunk":
        layer, p, faults = chunk(4, 2, 24, 16, SIZE, 4, 50.0, 1.0), "l0.mix.", ("chunk", "chunk_size")
        end = (place // SIZE + 1) * SIZE                      # the first position of the next chunk
        return layer, p, faults, [end - 1], [end, end + 1]
    if kind == "differential":
        layer, p, faults = diff(4, 2, 24, 16, SIZE, 4, 50.0, 1.0), "l0.mix.", ("window", "narrow")
        return layer, p, faults, [place + 1, place + SIZE - 1], [place + SIZE, place + SIZE + 1]
    layer, p, faults = pair(capped(4, 2, 24, 16, SIZE, 7, 20.0, 1.0)), "l0.mix.left.", ("window", "narrow", "keep", "keep_more")
    if place < 7:
        return layer, p, faults, [place + SIZE - 1, place + SIZE, place + 3 * SIZE], []
    return layer, p, faults, [place + 1, place + SIZE - 1], [place + SIZE, place + SIZE + 1]


EDGES = [(k, p) for k in ("chunk", "differential", "kept") for p in (31, 32, 63, 64, 89, 90)] + [("kept", p) for p in (0, 6, 7)] + [("chunk", 44), ("chunk", 45)]


def case_edge(tmp, device, dtype, kind, place):
    """One token's query is another token's key: it finds that token's one occurrence — at a page's border, the first or last kept
    token — while it is visible, and not from the next position on: in a prompt, across portions cut there, and decoded."""
    layer, p, faults, seeing, blind = _edge(kind, place)
    cfg = make_cfg([layer], width=64, scale=1.2)
    found, asking = 147, 148
    m = layer["mixer"].get("left", layer["mixer"])
    H, G, D, maps = m["heads"], m["kv_heads"], m["dim"], 2 if kind == "differential" else 1

    def edit(Wt):
        _silence("right.o")(Wt)
        for k in Wt:
            if k.endswith(("q.norm", "k.norm")):
                Wt[k] = Wt[k] * 0.0 + 1.0
        h = Wt["embed"] * 1.2
        q, k = Wt[p + "q"], Wt[p + "k"]
        aim = (q @ h[asking]).view(G, H // G, maps, D).clone()
        aim[:, :, 0] = (k @ h[found]).view(G, 1, maps, D)[:, :, 0]           # differential: the first map only
        Wt[p + "q"] = q + torch.outer(aim.reshape(-1) - q @ h[asking], h[asking]) / h[asking].square().sum()
    W, rig = _setup(tmp, cfg, dtype, device, seed=31, edit=edit)
    n = max(seeing + blind) + 6
    toks = [t % 140 for t in tokens(n, 140, 15)]
    toks[place] = found
    for a in seeing + blind:
        if a != place:
            toks[a] = asking
    want = expect(cfg, W, toks)
    changed = list(toks)
    changed[place] = 3
    other = expect(cfg, W, changed)
    for a in seeing:
        if a != place:
            assert rel_err(other[[a]], want[[a]]) > 2.5 * TOL[dtype], f"token {a} must see {place}"
    for a in blind:
        assert rel_err(other[[a]], want[[a]]) == 0.0, f"token {a} must not see {place}"
    rows = [a for a in seeing + blind if a != place]
    moved = max(rel_err(expect(cfg, W, toks, (f,))[rows], want[rows]) for f in faults)
    assert moved > 2.5 * TOL[dtype], moved
    last = rows[-1]
    for name, sizes in (("whole", [n]), ("cut before", [place or n, n]), ("cut behind", [place + 1, n]), ("cut at the asking token", [last, n]),
                        ("cut behind it", [last + 1, n]), ("two tokens before it", [max(last - 2, 1), 2, 2, n]), ("decoded", [max(place - 1, 1)] + [1] * n)):
        _check(rig.run({name: toks}, alone(name, n, sizes))[name], want, dtype, f"{kind}: key at {place}, {name}", single=True)
        _check(rig.run({name: changed}, alone(name, n, sizes))[name], other, dtype, f"{kind}: other key at {place}, {name}", single=True)


# ---------------------------------------------------------------- first tokens, very short requests, long decoding
def case_first_tokens_and_long_decode(tmp, device, dtype):
    W, rig = _setup(tmp, FULL, dtype, device, seed=15)
    for n in (1, 2, 3, 5):
        toks = tokens(n, FULL["vocab"], 30 + n)
        _check(rig.run({"x": toks}, alone("x", n, [1]))["x"], expect(FULL, W, toks), dtype, f"{n}-token request")
        _check(rig.run({"y": toks}, alone("y", n, [n]))["y"], expect(FULL, W, toks), dtype, f"{n}-token prompt")
    toks = tokens(190, FULL["vocab"], 5)
    _check(rig.run({"long": toks}, alone("long", 190, [20] + [1] * 170))["long"], expect(FULL, W, toks), dtype, "170 decoded tokens")


# ---------------------------------------------------------------- other sizes
def other_size_configs():
    return {
        # heads in multiples of 8 and 16: chunks on the tile kernel, single tokens on the heads-as-columns kernel
        "matrix-core shapes, eight heads on one key head":
            make_cfg([chunk(8, 1, 32, 48, 70, 16, mlp={"kind": "dense", "ff": 256, "limit": 3.0}), diff(16, 2, 24, 32, 41, 24),
                      pair(capped(8, 1, 40, 16, 50, 33, 6.0), delta(8, 4, 48, 64, 4), mlp={"kind": "dense", "ff": 128, "limit": 0.7}), again(1)],
                     width=128, vocab=90),
        "tiles, three heads on a key head": make_cfg(
            [diff(6, 2, 72, 80, 100, 36), chunk(3, 1, 104, 144, 33, 104), pair(capped(9, 3, 16, 32, 20, 40, 2.0), delta(3, 3, 20, 36, 2))], width=80, vocab=77),
        "all sizes odd": make_cfg(
            [pair(capped(9, 3, 17, 21, 13, 1, 2.5), delta(5, 1, 11, 9, 6), mlp={"kind": "dense", "ff": 37, "limit": 0.9}), diff(5, 5, 7, 11, 5, 6),
             chunk(3, 1, 13, 7, 11, 10), again(0)], width=50, vocab=131, eps=1e-3, scale=2.5),
        "one of everything": make_cfg(
            [chunk(1, 1, 4, 3, 1, 2), diff(1, 1, 4, 5, 1, 4), pair(capped(1, 1, 5, 3, 1, 1, 0.5), delta(1, 1, 4, 5, 1), (1.0, 1.0), mlp={"kind": "dense", "ff": 1, "limit": 1.0}),
             pair(capped(1, 1, 8, 8, 1, 0, 9.0), delta(4, 4, 8, 4, 1), mlp={"kind": "dense", "ff": 4, "limit": 5.0})], width=24, vocab=33, scale=1.0),
        # state rows past the block path (step kernel over whole chunks), and the widest that it takes; many heads
        "wide states, many heads": make_cfg(
            [pair(right=delta(2, 1, 200, 40, 4)), pair(right=delta(1, 1, 300, 70, 2)), pair(capped(16, 2, 16, 16, 64, 32, 4.0), delta(64, 8, 24, 33, 4))],
            width=64, vocab=70),
        "long filters, values wider than keys": make_cfg(
            [pair(capped(2, 2, 8, 96, 90, 20), delta(4, 2, 8, 96, 9)), diff(2, 1, 8, 120, 64, 2, lam=0.1), chunk(2, 2, 8, 136, 96, 6), pair(right=delta(2, 2, 96, 8, 12))],
            width=96, vocab=61),
    }


def case_other_sizes(tmp, device, dtype, name):
    cfg = other_size_configs()[name]
    W, rig = _setup(tmp, cfg, dtype, device, seed=17, ranks=(3, 5) if "odd" in name else (1, 1) if "one of" in name else (16, 8))
    toks = tokens(85, cfg["vocab"], 6)
    want = expect(cfg, W, toks)
    _check(rig.run({"w": toks}, alone("w", 85, [85]))["w"], want, dtype, name + " whole")
    _check(rig.run({"c": toks}, alone("c", 85, [2, 30, 1, 1, 33, 1]))["c"], want, dtype, name + " portions")
    if name.startswith(("matrix-core", "tiles")):             # tiles that start inside a page, with hundreds of keys behind them
        toks = tokens(300, cfg["vocab"], 8)
        want = expect(cfg, W, toks)
        _check(rig.run({"l": toks}, alone("l", 300, [45, 130, 17, 64, 43, 1]))["l"], want, dtype, name + " long portions")


# ---------------------------------------------------------------- greedy generation through the engine's own entry point
def case_generate(tmp, device, dtype, graphs=False):
    from dli_amd.config import CacheConfig, EngineConfig, SamplingParams, SchedulerConfig, resolve_model
    from dli_amd.engine.engine import LLMEngine
    W = write_checkpoint(tmp, FULL, 19, bf16=dtype == "bfloat16")
    mcfg, wpath = resolve_model(str(tmp), dtype)
    seqs, lens = (8, (5, 61, 30, 90, 2, 17, 33, 64, 1, 45, 8)) if graphs else (3, (5, 61, 30, 90, 2))
    eng = LLMEngine(EngineConfig(model=mcfg, weights_path=wpath, device=device, cache=CacheConfig(num_blocks=8 * seqs),
                                 sched=SchedulerConfig(max_num_seqs=seqs, max_num_batched_tokens=64, max_model_len=256,
                                                       long_prefill_chunk=40, token_alignment=0),
                                 use_hip_graphs=graphs, graph_batch_sizes=(1, 2, 4, 8), tune_gemms=False))
    if graphs:
        eng.warmup()
    prompts = [tokens(n, FULL["vocab"], 40 + n) for n in lens]                     # more requests than slots: some wait
    n_new = 10
    outs = eng.generate(None, SamplingParams(temperature=0.0, max_tokens=n_new, ignore_eos=True), prompt_ids=prompts)
    compared = 0
    for p, o in zip(prompts, outs):
        assert len(o) == n_new
        seq = list(p) + list(o)                                   # teacher-forced: every generated token is the oracle's argmax
        logits = oracle.forward(resolved(FULL), W, seq)[0]
        for j, tok in enumerate(o):
            row = logits[len(p) - 1 + j]
            top2 = torch.topk(row, 2).values
            if float(top2[0] - top2[1]) > (1e-3 if dtype == "float32" else 0.1) * float(row.std()):   # skip near-ties
                assert int(torch.argmax(row)) == tok
                compared += 1
    assert compared > len(lens) * n_new // 2
    assert eng.bm.num_free == eng.bm.num_blocks and eng.bm.num_free_state_slots == seqs
    if graphs:
        assert eng.runner.stats["graph_steps"] > 0, eng.runner.selftest
    return eng
