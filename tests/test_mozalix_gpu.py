"""Mozalix stacks on the gfx950 kernels (``csrc/kernels/postmix.hip``, the channel-decay recurrence of ``gatemix.hip`` and the extended
attention / convolution / activation kernels), fp32 and bf16, against the plain oracle: the cases of ``mozalix_cases`` on ``cuda``,
plus generation with captured decode / mixed-step hipGraphs and kernel-against-kernel and kernel-against-reference comparisons of
the fast paths."""
import pytest
import torch

import mozalix_cases as cases
import mozalix_oracle as oracle
from test_nefarax_gpu import _step

pytestmark = pytest.mark.gpu
DTYPES = ["float32", "bfloat16"]


@pytest.fixture(autouse=True)
def _needs_gpu():
    assert torch.cuda.is_available(), "GPU tests need a GPU"
    from dli_amd import ops
    ops.hip()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind", sorted(cases.MECHANISMS))
def test_each_mechanism_alone(tmp_path, kind, dtype):
    cases.case_mechanism(tmp_path, "cuda", dtype, kind)


@pytest.mark.parametrize("dtype", DTYPES)
def test_every_piece_shows_when_wrong(tmp_path, dtype):
    cases.case_each_piece_matters(tmp_path, "cuda", dtype)


@pytest.mark.parametrize("dtype", DTYPES)
def test_prefill_decode_and_portions(tmp_path, dtype):
    cases.case_prefill_decode_portions(tmp_path, "cuda", dtype)


@pytest.mark.parametrize("dtype", DTYPES)
def test_unequal_requests_in_one_batch(tmp_path, dtype):
    cases.case_mixed_batch(tmp_path, "cuda", dtype)


@pytest.mark.parametrize("dtype", DTYPES)
def test_chunks_beside_single_tokens_at_matrix_core_sizes(tmp_path, dtype):
    cases.case_mixed_batch_on_tiles(tmp_path, "cuda", dtype)


@pytest.mark.parametrize("dtype", DTYPES)
def test_pages_and_slots_used_again(tmp_path, dtype):
    cases.case_reuse(tmp_path, "cuda", dtype)


def test_far_tokens(tmp_path):
    cases.case_far_token(tmp_path, "cuda", "float32")          # the effect of one far token is below bf16 rounding


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind,place", cases.EDGES)
def test_keys_at_edges(tmp_path, kind, place, dtype):
    cases.case_edge(tmp_path, "cuda", dtype, kind, place)


def test_first_tokens_and_long_decoding(tmp_path):
    cases.case_first_tokens_and_long_decode(tmp_path, "cuda", "float32")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(cases.other_size_configs()))
def test_other_sizes(tmp_path, name, dtype):
    cases.case_other_sizes(tmp_path, "cuda", dtype, name)


@pytest.mark.parametrize("dtype", DTYPES)
def test_greedy_generation_eager(tmp_path, dtype):
    cases.case_generate(tmp_path, "cuda", dtype)


@pytest.mark.parametrize("dtype", DTYPES)
def test_greedy_generation_with_hip_graphs(tmp_path, dtype):
    eng = cases.case_generate(tmp_path, "cuda", dtype, graphs=True)
    st = eng.runner.selftest
    assert st.get("graph_vs_eager", {}).get("ok", True) and st.get("mixed_graph_vs_eager", {}).get("ok", True), st


def test_block_scan_against_the_step_kernel(tmp_path, monkeypatch):
    """A recurrence over a long prompt: blocks on the matrix cores against the token-by-token walk of the step kernel."""
    import numpy as np
    from dli_amd.ops import seqmix
    cfg = cases.MEMORY

    def edit(Wt):
        cases._remember(Wt)
        cases._silence("left.o")(Wt)
    W, rig = cases._setup(tmp_path, cfg, "float32", "cuda", seed=27, edit=edit)
    toks = cases.tokens(400, cfg["vocab"], 11)
    blocks = rig.run({"a": toks}, cases.alone("a", 400, [333, 67]))["a"]
    monkeypatch.setattr(seqmix, "BLOCK_SCAN", False)
    walk = rig.run({"b": toks}, cases.alone("b", 400, [333, 67]))["b"]
    assert not np.array_equal(blocks, walk), "both runs took the same kernel"
    cases._check(blocks, walk, "float32", "blocks against the walk")
    cases._check(blocks, cases.expect(cfg, W, toks), "float32", "blocks against the oracle")


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H,G,D,Dv", [(4, 2, 64, 48), (2, 2, 128, 128), (3, 1, 30, 17), (1, 1, 256, 16), (6, 3, 100, 64), (64, 8, 32, 40), (2, 1, 280, 24)])
def test_channel_scan_kernels_against_the_reference(H, G, D, Dv, dtype):
    """Single tokens and chunks of several sequences in one launch, twice in a row (the second step carries the states), with decays
    from almost none to e^-30 per token side by side in one block and one head, and the state slots shuffled."""
    from dli_amd.ops import seqmix
    torch.manual_seed(3)
    state_g = None
    starts = [0, 7, 0, 0, 0]
    rate, bias = torch.rand(H) + 0.1, torch.randn(H * D)
    for lens in ([1, 1, 2, 65, 190], [1, 64, 1, 3, 129]):
        mc, T = _step(lens, starts, "cpu")
        mg, _ = _step(lens, starts, "cuda")
        slots = int(max(mc.state_slots)) + 1
        if state_g is None:
            state_c = torch.randn(slots, H, D, Dv) * 0.3
            state_g = state_c.cuda()
        q, v = torch.randn(T, G * D) * D ** -0.5, torch.randn(T, H * Dv)
        k = torch.nn.functional.normalize(torch.randn(T, G, D), dim=-1).view(T, G * D)
        z = torch.empty(T, H * D).uniform_(-12.0, 6.0)
        z[torch.rand(T, H * D) < 0.02] = 30.0                  # a channel forgets everything, inside a block
        z = z.to(dtype)
        weight = torch.rand(T, H)
        want = seqmix.channel_delta_scan(q, k, v, z, rate, bias, weight, state_c, mc, H, G, D, Dv)
        wide = torch.zeros(T, H * D + 8, dtype=dtype, device="cuda")
        wide[:, :H * D] = z.cuda()
        got = seqmix.channel_delta_scan(q.cuda(), k.cuda(), v.cuda(), wide[:, :H * D], rate.cuda(), bias.cuda(), weight.cuda(), state_g, mg, H, G, D, Dv)
        scale = max(float(want.abs().max()), 1.0)
        assert float((got.cpu() - want).abs().max()) < 2e-5 * scale
        assert float((state_g.cpu() - state_c).abs().max()) < 2e-5 * max(float(state_c.abs().max()), 1.0)
        starts = [s + n for s, n in zip(starts, lens)]


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("W", [256, 90, 4100])
def test_norm_and_activation_kernels_against_the_reference(W, dtype):
    from dli_amd.ops import seqmix
    torch.manual_seed(6)
    T = 37
    tol = dict(rtol=1e-5, atol=1e-5) if dtype == torch.float32 else dict(rtol=1e-2, atol=1e-2)
    x, w, w2 = torch.randn(T, W), torch.randn(W), torch.randn(W)
    for size in (1.0, 1e-3):                                   # at and below the norm's epsilon
        y = (torch.randn(T, W) * size).to(dtype)
        for last in (None, w2):
            xc, xg = x.clone(), x.cuda()
            want = seqmix.post_norm_add(xc, y, w, 1e-4, dtype, last)
            got = seqmix.post_norm_add(xg, y.cuda(), w.cuda(), 1e-4, dtype, last.cuda() if last is not None else None)
            assert torch.allclose(xg.cpu(), xc, rtol=1e-5, atol=1e-5) and torch.allclose(got.cpu().float(), want.float(), **tol)
    table, ids = torch.randn(50, W).to(dtype), torch.randint(0, 50, (T,), dtype=torch.int32)
    want, got = seqmix.embed_rows(ids, table, 0.3, dtype), seqmix.embed_rows(ids.cuda(), table.cuda(), 0.3, dtype)
    assert all(torch.allclose(a.cpu().float(), b.float(), **tol) for a, b in zip(got, want)) and got[1].dtype == dtype
    gu = (torch.randn(T, 2 * W) * 4).to(dtype)
    assert torch.allclose(seqmix.act_mul(gu.cuda(), "clamped", 1.7).cpu().float(), seqmix.act_mul(gu, "clamped", 1.7).float(), **tol)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H,G,D,Dv,dims,maps", [(6, 2, 64, 32, 64, 1), (4, 4, 128, 128, 32, 1), (6, 3, 24, 16, 8, 2), (4, 1, 30, 21, 12, 2), (2, 1, 256, 8, 0, 1), (5, 5, 7, 3, 2, 1)])
def test_head_norm_kernel_against_the_reference(H, G, D, Dv, dims, maps, dtype):
    from dli_amd.ops import seqmix
    torch.manual_seed(7)
    T = 29
    cols = (H + G) * maps * D + G * Dv
    proj = torch.randn(T, cols + 8).to(dtype)
    pos = torch.randint(0, 200000, (T,), dtype=torch.int32)
    slots = torch.randperm(96)[:T].int()
    slots[5] = -1
    freq = seqmix.rotary_inv_freq(7000.0, dims)
    tol = dict(rtol=1e-4, atol=1e-4) if dtype == torch.float32 else dict(rtol=2e-2, atol=2e-2)
    for qw, kw in ((torch.randn(D), torch.randn(D)), (None, None)):
        c = [torch.zeros(3, 32, G * maps * D, dtype=dtype), torch.zeros(3, 32, G * Dv, dtype=dtype)]
        g = [t.cuda() for t in c]
        cu = lambda t: t.cuda() if t is not None else None
        want = seqmix.head_norm_rope_cache(proj[:, :cols], qw, kw, 1e-4, pos, freq, dims, slots, *c, H, G, D, Dv, maps)
        got = seqmix.head_norm_rope_cache(proj.cuda()[:, :cols], cu(qw), cu(kw), 1e-4, pos.cuda(), freq.cuda(), dims, slots.cuda(), *g, H, G, D, Dv, maps)
        for a, b in zip([got, *g], [want, *c]):
            assert torch.allclose(a.cpu().float(), b.float(), **tol)


def _attention_step(starts, lens, device):
    """Step metadata with pages: sequence ``i`` owns pages ``i, i + B, i + 2B, …`` of the cache."""
    m, T = _step(lens, starts, device)
    order = sorted(range(len(lens)), key=lambda i: lens[i] != 1)
    B = len(lens)
    m.block_tables = torch.tensor([[i + B * j for j in range(16)] for i in order], dtype=torch.int32, device=device)
    m.seq_lens = torch.tensor([starts[i] + lens[i] for i in order], dtype=torch.int32, device=device)
    m.counts_on_device = False
    return m, T


ATTENTION = {
    "chunk, sink": (8, 2, 64, 80, dict(chunk=75), True), "chunk of one": (4, 4, 32, 16, dict(chunk=1), True), "kept tokens, cap": (8, 1, 48, 32, dict(window=40, keep_first=6, cap=3.0), False),
    "kept pages, cap": (16, 1, 40, 64, dict(window=33, keep_first=70, cap=20.0), False), "kept only": (3, 1, 16, 48, dict(window=1, keep_first=33, cap=1.0), False),
    "wide": (4, 2, 200, 208, dict(window=100, keep_first=3, cap=5.0), False), "long chunk": (6, 2, 104, 144, dict(chunk=160), True)}


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("name", sorted(ATTENTION))
def test_masked_attention_kernels_against_the_reference(name, dtype):
    """Chunks and single tokens of several sequences: the tile, heads-as-columns and per-token kernels, with fp32 results too."""
    from dli_amd.ops import seqmix
    H, G, D, Dv, kw, has_sink = ATTENTION[name]
    torch.manual_seed(8)
    lens, starts = [1, 1, 2, 70, 131, 33], [300, 0, 64, 150, 0, 95]
    mc, T = _attention_step(starts, lens, "cpu")
    mg, _ = _attention_step(starts, lens, "cuda")
    kc, vc = torch.randn(96, 32, G * D).to(dtype), torch.randn(96, 32, G * Dv).to(dtype)
    q = (torch.randn(T, H, D) * 1.5).to(dtype)
    sink = torch.randn(H) + 1.0 if has_sink else None
    want = seqmix.token_attention(torch.zeros(T, H, Dv), q.float(), None, kc.float(), vc.float(), mc, G, Dv, D ** -0.5, sink=sink, out_scale=0.6, **kw)
    tol = 3e-5 if dtype == torch.float32 else 2e-2
    for out_dtype in {dtype, torch.float32}:
        got = seqmix.token_attention(torch.zeros(T, H, Dv, dtype=out_dtype, device="cuda"), q.cuda(), None, kc.cuda(), vc.cuda(), mg, G, Dv, D ** -0.5,
                                     sink=sink.cuda() if has_sink else None, out_scale=0.6, **kw)
        err = (got.cpu().float() - want).abs().max()
        assert float(err) < (3e-4 if out_dtype == torch.float32 else tol) * max(float(want.abs().max()), 1.0), float(err)
        if dtype == torch.bfloat16:                            # the per-token kernel on the same rows
            slow = torch.zeros(T, H, Dv, dtype=out_dtype, device="cuda")
            seqmix._attend_rows(seqmix._hip(), slow, q.cuda(), None, kc.cuda(), vc.cuda(), mg, -1, (G, Dv, D ** -0.5, kw.get("window", 0), None, None, None),
                                (None, sink.cuda() if has_sink else None, kw.get("chunk", 0), kw.get("keep_first", 0), kw.get("cap", 0.0), G, 0.6))
            assert float((slow.cpu().float() - got.cpu().float()).abs().max()) < (3e-4 if out_dtype == torch.float32 else tol)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H,G,D,Dv,window", [(8, 2, 64, 80, 50), (8, 1, 24, 32, 33), (3, 1, 128, 128, 200), (4, 4, 200, 208, 70), (6, 2, 20, 12, 9), (16, 2, 32, 256, 40)])
def test_differential_attention_kernels_against_the_reference(H, G, D, Dv, window, dtype):
    """Both maps, their difference and its norm: one kernel over prefill tiles, per-token / heads-as-columns kernels elsewhere."""
    from dli_amd.ops import seqmix
    torch.manual_seed(9)
    kc, vc = torch.randn(96, 32, G * 2 * D).to(dtype), torch.randn(96, 32, G * Dv).to(dtype)
    lam = torch.tensor([0.7])
    for lens, starts in (([1, 1, 2, 70, 131, 33], [300, 0, 64, 150, 0, 95]), ([64, 64], [0, 40]), ([1, 1, 1], [0, 31, 400])):
        mc, T = _attention_step(starts, lens, "cpu")
        mg, _ = _attention_step(starts, lens, "cuda")
        q = (torch.randn(T, 2 * H, D) * 1.5).to(dtype)
        want = torch.zeros(T, H * Dv)
        seqmix.map_attention(want, q.float(), kc.float(), vc.float(), mc, G, Dv, D ** -0.5, window, lam, 1e-5, 0.8)
        buf = torch.full((T, H * Dv + 8), 3.0, dtype=dtype, device="cuda")
        seqmix.map_attention(buf[:, :H * Dv], q.cuda(), kc.cuda(), vc.cuda(), mg, G, Dv, D ** -0.5, window, lam.cuda(), 1e-5, 0.8)
        got = buf[:, :H * Dv].cpu().float()
        assert float((got - want).abs().max()) < (1e-4 if dtype == torch.float32 else 3e-2) * max(float(want.abs().max()), 1.0)
        assert float((buf[:, H * Dv:] - 3.0).abs().max()) == 0.0
    assert oracle.F64 == torch.float64


def test_generation_at_layer_sizes_of_a_real_model():
    """Random weights, heads of 128, hipGraph decode steps: the start-up self-test compares captured steps with eager ones."""
    from dli_amd.config import CacheConfig, EngineConfig, SamplingParams, SchedulerConfig, mozalix_config
    from dli_amd.engine.engine import LLMEngine
    ff = {"kind": "dense", "ff": 1408, "limit": 7.0}
    layers = [cases.chunk(8, 2, 128, 128, 192, 64, 1e5, 128 ** -0.5, ff), cases.diff(8, 2, 64, 128, 128, 64, 1e5, 0.125, 0.5, ff),
              cases.pair(dict(cases.capped(8, 1, 128, 64, 128, 4, 30.0, 0.09)), dict(cases.delta(8, 4, 128, 128, 4), lora=64, gate_lora=64), mlp=ff), cases.again(0)]
    eng = LLMEngine(EngineConfig(model=mozalix_config(cases.make_cfg(layers, width=1024, vocab=2000)), device="cuda", cache=CacheConfig(num_blocks=256),
                                 sched=SchedulerConfig(max_num_seqs=8, max_num_batched_tokens=512, max_model_len=700, token_alignment=0),
                                 use_hip_graphs=True, graph_batch_sizes=(1, 4, 8), tune_gemms=False))
    eng.warmup()
    st = eng.runner.selftest
    assert st.get("graph_vs_eager", {}).get("ok", True) and st.get("mixed_graph_vs_eager", {}).get("ok", True), st
    outs = eng.generate(None, SamplingParams(temperature=0.0, max_tokens=20, ignore_eos=True), prompt_ids=[cases.tokens(n, 2000, n) for n in (3, 500, 190, 260, 64)])
    assert all(len(o) == 20 for o in outs) and eng.runner.stats["graph_steps"] > 0
