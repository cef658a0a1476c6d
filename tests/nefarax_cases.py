"""The Nefarax test cases, parametrised by device and dtype.  Each case builds its own small configuration, writes a
checkpoint from the plain oracle's random weights (``nefarax_oracle``), replays step schedules through the engine
(``rodelix_common.Rig``: the engine's runner, block manager, cache, state slots and kernels) and compares every position's
logits with the oracle.  The same cases run on the CPU path (``test_nefarax.py``) and on the GPU kernels
(``test_nefarax_gpu.py``)."""
from __future__ import annotations

import copy
import json
import os

import numpy as np
import torch

import nefarax_oracle as oracle
from rodelix_common import Rig, TOL, alone, chunks, rel_err, tokens

DENSE = {"kind": "dense", "ff": 88}
BANDS = {"factor": 4.0, "high": 8.0, "low": 2.0, "original": 96}


def delta(heads=6, kv_heads=2, dim=12, vdim=20, conv=3, mlp=None):
    return {"type": "delta", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}, "mlp": copy.deepcopy(mlp)}


def mlstm(heads=3, dim=16, vdim=24, gate_cap=6.0, mlp=None):
    return {"type": "mlstm", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": gate_cap}, "mlp": copy.deepcopy(mlp)}


def attn(heads=6, kv_heads=3, dim=20, conv=4, scale=0.3, dims=12, base=3000.0, scaling=BANDS):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "conv": conv, "scale": scale}
    if dims:
        m["rot"] = {"base": base, "dims": dims}
        if scaling:
            m["rot"]["scaling"] = dict(scaling)
    return m


def ssd(heads=6, vdim=12, state=20, groups=3, conv=3, norm_groups=4):
    return {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "conv": conv, "norm_groups": norm_groups}


def pair(left=None, right=None, mlp=None):
    return {"type": "parallel", "mixer": {"left": left or attn(), "right": right or ssd()}, "mlp": copy.deepcopy(mlp)}


def make_cfg(layers, width=72, vocab=149, mult=0.6, eps=1e-5):
    return {"architecture": "Nefarax", "vocab": vocab, "width": width, "residual_mult": mult, "norm": {"eps": eps},
            "layers": [copy.deepcopy(l) for l in layers]}


# every mixer, with and without a feed-forward, two of each with sizes of their own
FULL = make_cfg([mlstm(gate_cap=4.0, mlp=DENSE), delta(mlp=DENSE), pair(mlp=DENSE), delta(heads=4, kv_heads=4, dim=16, vdim=8, conv=5),
                 pair(attn(heads=4, kv_heads=1, dim=16, conv=2, dims=16, scaling=None), ssd(heads=4, vdim=10, state=16, groups=1, conv=5, norm_groups=2)),
                 mlstm(heads=2, dim=24, vdim=16, gate_cap=12.0)])


def write_checkpoint(path, cfg, seed=0, bf16=False, edit=None):
    """config.json + model.safetensors; returns the weights as stored (fp32 values) for the oracle."""
    from safetensors.torch import save_file
    os.makedirs(path, exist_ok=True)
    W = oracle.random_weights(cfg, seed)
    if edit:
        edit(W)
    if bf16:
        W = {k: v.to(torch.bfloat16) for k, v in W.items()}
    with open(os.path.join(path, "config.json"), "w") as fh:
        json.dump(cfg, fh)
    save_file({k: v.contiguous() for k, v in W.items()}, os.path.join(path, "model.safetensors"))
    return {k: v.float() for k, v in W.items()}


def expect(cfg, W, toks, faults=()):
    return oracle.forward(cfg, W, toks, faults)[0].numpy()


def _setup(tmp, cfg, dtype, device, seed=0, edit=None, **rig):
    W = write_checkpoint(tmp, cfg, seed, bf16=dtype == "bfloat16", edit=edit)
    return W, Rig(tmp, dtype, device, **rig)


def _check(got, want, dtype, what=""):
    e = rel_err(got, want)
    assert e < TOL[dtype], f"{what}: relative error {e:.3e} over {TOL[dtype]:.1e}"


# ---------------------------------------------------------------- each mechanism alone
def _silence(*ends):
    def edit(Wt):
        for k in Wt:
            if k.endswith(ends):
                Wt[k] = Wt[k] * 0.0
    return edit


MECHANISMS = {
    "delta rule": (make_cfg([delta(), delta(heads=2, kv_heads=1, dim=24, vdim=16, conv=1)]), None),
    "mlstm": (make_cfg([mlstm(), mlstm(heads=1, dim=8, vdim=40, gate_cap=3.0)]), None),
    "attention half": (make_cfg([pair(), pair(attn(dims=8, scaling=None))]), _silence("right.out")),
    "attention half without rotation": (make_cfg([pair(attn(dims=0)), pair(attn(heads=3, conv=1, dims=0))]), _silence("right.out")),
    "state-space half": (make_cfg([pair(), pair(right=ssd(heads=2, groups=1, norm_groups=1))]), _silence("left.out")),
    "normed pair": (make_cfg([pair(), pair()]), None),
    "feed-forward": (make_cfg([delta(mlp=DENSE), pair(mlp=DENSE), mlstm(mlp=DENSE)]), _silence("mix.o", "left.out", "right.out")),
    "feed-forward beside its mixer": (make_cfg([delta(mlp=DENSE), mlstm(mlp=DENSE)], mult=1.0), None),
}


def case_mechanism(tmp, device, dtype, kind):
    cfg, edit = MECHANISMS[kind]
    W, rig = _setup(tmp, cfg, dtype, device, seed=3, edit=edit)
    toks = tokens(150, cfg["vocab"], 1)
    want = expect(cfg, W, toks)
    _check(rig.run({"a": toks}, alone("a", len(toks), [len(toks)]))["a"], want, dtype, f"{kind} whole prompt")
    _check(rig.run({"b": toks}, alone("b", len(toks), [31, 2, 1, 40, 1, 1, 7]))["b"], want, dtype, f"{kind} in portions")


# ---------------------------------------------------------------- getting a mechanism wrong must show
FAULTS = ("squash", "norm_bias", "mult", "stale", "conv", "conv_act", "unit", "beta", "decay", "erase", "late_read", "out_norm", "gate",
          "cap", "normaliser", "rotated_values", "scaling", "rotation", "sink", "skip", "late_gate", "one_group", "dt_bias",
          "half", "side_norm")


def _telling(Wt):
    """Weights under which every single mistake moves the logits: small divisors matter (outputs near the norm's epsilon),
    strong gates, peaked scores with a heavy sink."""
    for k in list(Wt):
        if k.endswith("left.sink"):
            Wt[k] = Wt[k] + 2.0
        if k.endswith("right.conv.b"):
            Wt[k] = Wt[k] * 3.0
        if k.endswith(("mix.i", "mix.f")):
            Wt[k] = Wt[k] * 4.0
        if k.endswith("mix.v") and f"{k[:-1]}i" in Wt:
            Wt[k] = Wt[k] * 0.05


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
                        ("block edges", [63, 2, 65, 5]), ("shorter than the convolutions", [2, 1, 2, 2, 1, 1, 3, 88])):
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
    # one-token prompts in slots whose last owner left states, convolution inputs and running maxima behind
    singles = {f"s{j}": tokens(4, FULL["vocab"], 30 + j) for j in range(3)}
    got = rig.run(singles, [[("s0", 1), ("s1", 1)], [("s0", 1), ("s1", 3)], [("s0", 2)], [("s2", 1)], [("s2", 1)], [("s2", 2)]])
    for i in singles:
        _check(got[i], expect(FULL, W, singles[i]), dtype, f"request {i} starting with one token")
    bm = rig.rep.bm
    assert bm.num_free == bm.num_blocks and bm.num_free_state_slots == 2


# ---------------------------------------------------------------- a token far back; memory of the recurrences
def _remember(Wt):
    """Slow decays, and for the attention scores that let single keys stand out."""
    for k in list(Wt):
        if k.endswith("A_log"):
            Wt[k] = Wt[k] - 5.0                               # states remember hundreds of tokens
        if k.endswith("dt_bias") and "right" not in k:
            Wt[k] = Wt[k] - 2.0
        if k.endswith("mix.f.b"):
            Wt[k] = Wt[k] + 6.0
        if k.endswith("mix.f"):
            Wt[k] = Wt[k] * 0.2
        if k.endswith(("left.q", "left.k")):
            Wt[k] = Wt[k] * 1.6
        if k.endswith("left.sink"):
            Wt[k] = Wt[k] - 2.0


FAR = {
    "delta rule": (make_cfg([delta(dim=32, vdim=24), delta(dim=40, vdim=16)], width=64), ()),
    "mlstm": (make_cfg([mlstm(gate_cap=15.0), mlstm(gate_cap=15.0)], width=64), ()),
    "attention half": (make_cfg([pair(), pair()], width=64), ("right.out",)),
    "state-space half": (make_cfg([pair(), pair()], width=64), ("left.out",)),
}


def case_far_token(tmp, device, dtype, which):
    cfg, quiet = FAR[which]

    def edit(Wt):
        _remember(Wt)
        if quiet:
            _silence(*quiet)(Wt)
    W, rig = _setup(tmp, cfg, dtype, device, seed=13, edit=edit)
    toks = tokens(330, cfg["vocab"], 4)
    want = expect(cfg, W, toks)
    changed = list(toks)
    changed[1] = (toks[1] + 17) % cfg["vocab"]                # position 1 must reach the last rows
    assert rel_err(expect(cfg, W, changed)[-20:], want[-20:]) > 5 * TOL[dtype], which
    _check(rig.run({"p": toks}, alone("p", 330, [300] + [1] * 30))["p"], want, dtype, f"far token ({which}), prompt then decoding")
    _check(rig.run({"c": toks}, alone("c", 330, [64, 63, 2, 129]))["c"], want, dtype, f"far token ({which}), portions")


# ---------------------------------------------------------------- one key at a page's border
def case_page_border(tmp, device, dtype, place):
    """One token's query is another token's key: it finds that token's one occurrence, which sits at a page's border, among many
    others — in a prompt, across portions cut there, and decoded."""
    left = attn(heads=4, kv_heads=2, dim=24, conv=3, scale=0.8, dims=8, base=50.0, scaling=None)
    cfg = make_cfg([pair(left)], width=64)
    found, asking = 147, 148

    def edit(Wt):
        _silence("right.out")(Wt)
        p = "l0.mix.left."
        for c in ("q.conv", "k.conv"):                        # the token itself, next to nothing of the ones before
            Wt[p + c] = Wt[p + c] * 0.05
            Wt[p + c][:, -1] = 1.0
        h = oracle.tanh_norm(Wt["embed"], Wt["l0.norm1.alpha"], Wt["l0.norm1"], Wt["l0.norm1.b"])
        q, k = Wt[p + "q"] * 0.1, Wt[p + "k"]
        want = 2.0 * (k @ h[found]).view(2, 1, 24).expand(2, 2, 24).reshape(96)
        Wt[p + "q"] = q + torch.outer(want - q @ h[asking], h[asking]) / h[asking].square().sum()
    W, rig = _setup(tmp, cfg, dtype, device, seed=31, edit=edit)
    n = place + 90
    toks = [t % 140 for t in tokens(n, 140, 15)]
    toks[place] = found
    for a in (n - 1, n - 2, place + 33):
        toks[a] = asking
    want = expect(cfg, W, toks)
    changed = list(toks)
    changed[place] = 3
    moved = rel_err(expect(cfg, W, changed)[[place + 33]], want[[place + 33]])
    assert moved > 2.5 * TOL[dtype], moved
    for name, sizes in (("whole", [n]), ("cut before", [place, n - place]), ("cut behind", [place + 1, n - place - 1]),
                        ("decoded", [place - 1] + [1] * 40 + [n]), ("asked by decoding", [place + 30] + [1] * 60)):
        _check(rig.run({name: toks}, alone(name, n, sizes))[name], want, dtype, f"key at {place}, {name}")
        _check(rig.run({name: changed}, alone(name, n, sizes))[name], expect(cfg, W, changed), dtype, f"other key at {place}, {name}")


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
            make_cfg([pair(attn(8, 1, 32, 4, 0.2, 32), ssd(8, 32, 48, 2, 4, 8), mlp={"kind": "dense", "ff": 256}),
                      delta(8, 8, 48, 64, 4, mlp={"kind": "dense", "ff": 128}), mlstm(4, 64, 128, 15.0, mlp={"kind": "dense", "ff": 192})],
                     width=128, vocab=90),
        "all sizes odd": make_cfg(
            [delta(3, 1, 17, 21, 6, mlp={"kind": "dense", "ff": 37}), mlstm(5, 10, 7, 2.5), pair(attn(9, 3, 14, 3, 0.4, 6), ssd(5, 9, 11, 5, 2, 3)),
             delta(5, 5, 9, 33, 2)], width=50, vocab=131, eps=1e-3, mult=0.35),
        "one of everything": make_cfg(
            [delta(1, 1, 1, 1, 1), mlstm(1, 1, 1, 1.0), pair(attn(1, 1, 2, 1, 1.0, 2, scaling=None), ssd(1, 1, 1, 1, 1, 1)), delta(1, 1, 4, 8, 1),
             pair(attn(1, 1, 8, 1, 1.0, 0), ssd(4, 4, 4, 4, 1, 4), mlp={"kind": "dense", "ff": 1})], width=20, vocab=33, mult=1.0),
        # state rows past the block path (step kernel over whole chunks), and the widest that it takes; 64 state-space heads
        "wide states, many heads": make_cfg(
            [delta(2, 1, 200, 40, 4), mlstm(1, 300, 70, 15.0), mlstm(2, 130, 18, 15.0), pair(attn(4, 2, 16, 4, 0.2, 16), ssd(64, 33, 24, 2, 4, 11))],
            width=64, vocab=70),
        "long filters, values wider than keys": make_cfg(
            [delta(4, 2, 8, 96, 9), pair(attn(2, 2, 40, 7, 0.15, 24), ssd(3, 64, 8, 1, 8, 1)), delta(2, 2, 96, 8, 12)], width=96, vocab=61),
    }


def case_other_sizes(tmp, device, dtype, name):
    cfg = other_size_configs()[name]
    W, rig = _setup(tmp, cfg, dtype, device, seed=17)
    toks = tokens(85, cfg["vocab"], 6)
    want = expect(cfg, W, toks)
    _check(rig.run({"w": toks}, alone("w", 85, [85]))["w"], want, dtype, name + " whole")
    _check(rig.run({"c": toks}, alone("c", 85, [2, 30, 1, 1, 33, 1]))["c"], want, dtype, name + " portions")
    if name.startswith("matrix-core"):                        # tiles that start inside a page, with hundreds of keys behind them
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
    for p, o in zip(prompts, outs):
        assert len(o) == n_new
        seq = list(p) + list(o)                                   # teacher-forced: every generated token is the oracle's argmax
        logits = oracle.forward(FULL, W, seq)[0]
        for j, tok in enumerate(o):
            row = logits[len(p) - 1 + j]
            top2 = torch.topk(row, 2).values
            if float(top2[0] - top2[1]) > (1e-3 if dtype == "float32" else 0.05) * float(row.std()):   # skip near-ties
                assert int(torch.argmax(row)) == tok
    assert eng.bm.num_free == eng.bm.num_blocks and eng.bm.num_free_state_slots == seqs
    if graphs:
        assert eng.runner.stats["graph_steps"] > 0, eng.runner.selftest
    return eng
