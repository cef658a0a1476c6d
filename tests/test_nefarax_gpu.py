"""Nefarax stacks on the gfx950 kernels (``csrc/kernels/gatemix.hip`` and the extended convolution / norm / attention kernels),
fp32 and bf16, against the plain oracle: the cases of ``nefarax_cases`` on ``cuda``, plus generation with captured decode /
mixed-step hipGraphs and kernel-against-kernel and kernel-against-reference comparisons of the fast paths."""
import types

import pytest
import torch

import nefarax_cases as cases

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


@pytest.mark.parametrize("which", sorted(cases.FAR))
def test_far_tokens(tmp_path, which):
    cases.case_far_token(tmp_path, "cuda", "float32", which)   # the effect of one far token is below bf16 rounding


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("place", [31, 32, 63])
def test_keys_at_page_borders(tmp_path, place, dtype):
    cases.case_page_border(tmp_path, "cuda", dtype, place)


def test_first_tokens_and_long_decoding(tmp_path):
    cases.case_first_tokens_and_long_decode(tmp_path, "cuda", "float32")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(cases.other_size_configs()))
def test_other_sizes(tmp_path, name, dtype):
    if name == "one of everything" and dtype == "bfloat16":
        pytest.skip("vectors of one entry at unit length or unit RMS are signs of rounded numbers: compared in fp32 only")
    cases.case_other_sizes(tmp_path, "cuda", dtype, name)


@pytest.mark.parametrize("dtype", DTYPES)
def test_greedy_generation_eager(tmp_path, dtype):
    cases.case_generate(tmp_path, "cuda", dtype)


@pytest.mark.parametrize("dtype", DTYPES)
def test_greedy_generation_with_hip_graphs(tmp_path, dtype):
    eng = cases.case_generate(tmp_path, "cuda", dtype, graphs=True)
    st = eng.runner.selftest
    assert st.get("graph_vs_eager", {}).get("ok", True) and st.get("mixed_graph_vs_eager", {}).get("ok", True), st


@pytest.mark.parametrize("which", ["delta rule", "mlstm", "state-space half"])
def test_block_scan_against_the_step_kernel(tmp_path, monkeypatch, which):
    """A recurrence over a long prompt: blocks on the matrix cores against the token-by-token walk of the step kernel."""
    import numpy as np
    from dli_amd.ops import seqmix
    from rodelix_common import alone, tokens
    cfg, _ = cases.FAR[which]
    W, rig = cases._setup(tmp_path, cfg, "float32", "cuda", seed=27, edit=cases._remember)
    toks = tokens(400, cfg["vocab"], 11)
    blocks = rig.run({"a": toks}, alone("a", 400, [333, 67]))["a"]
    monkeypatch.setattr(seqmix, "BLOCK_SCAN", False)
    walk = rig.run({"b": toks}, alone("b", 400, [333, 67]))["b"]
    assert not np.array_equal(blocks, walk), "both runs took the same kernel"
    cases._check(blocks, walk, "float32", "blocks against the walk")
    cases._check(blocks, cases.expect(cfg, W, toks), "float32", "blocks against the oracle")


def _step(lens, starts, device):
    """Step metadata of sequences bringing ``lens`` tokens from positions ``starts``: single tokens first, then chunks (as the
    runner lays a step out), each in a state slot of its own."""
    import numpy as np
    from dli_amd import ops
    order = sorted(range(len(lens)), key=lambda i: lens[i] != 1)
    slot = [(3 * i + 2) % (len(lens) + 3) if (len(lens) + 3) % 3 else i + 1 for i in range(len(lens))]     # a sequence keeps its slot
    n = np.asarray([lens[i] for i in order], dtype=np.int32)
    p0 = [starts[i] for i in order]
    nd, T = int((n == 1).sum()), int(n.sum())
    qsl = np.concatenate([[0], np.cumsum(n)]).astype(np.int32)
    pos = np.concatenate([np.arange(p, p + c) for p, c in zip(p0, n)]).astype(np.int32)
    ts, tq = ops.build_prefill_tiles(n[nd:], nd, 64, (np.asarray(p0) + n)[nd:].astype(np.int32)) if nd < len(n) else (np.zeros(0), np.zeros(0))
    t = lambda a: torch.as_tensor(np.asarray(a, dtype=np.int32)).to(device)
    return types.SimpleNamespace(num_decode=nd, num_prefill=len(n) - nd, positions=t(pos), query_start_loc=t(qsl), num_seqs=len(n),
                                 token_seq=t(np.repeat(np.arange(len(n)), n)), state_slots=t([slot[i] for i in order]), counts=t([0, 0, len(ts), len(n)]), prefill_tile_seq=t(ts),
                                 prefill_tile_q0=t(tq), num_prefill_tiles=len(ts)), T


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("delta,normaliser,H,G,D,Dv", [(True, False, 4, 2, 64, 48), (True, False, 2, 2, 128, 128), (True, False, 3, 1, 30, 17),
                                                       (True, False, 1, 1, 256, 16), (False, True, 4, 4, 64, 64), (False, True, 2, 2, 21, 33),
                                                       (False, False, 64, 4, 48, 40), (False, False, 6, 2, 180, 64), (True, False, 64, 8, 32, 40)])
def test_scan_kernels_against_the_reference(delta, normaliser, H, G, D, Dv, dtype):
    """Single tokens and chunks of several sequences in one launch, twice in a row (the second step carries the states), with log
    decays from almost none to -20 inside one block (sums of hundreds, differences that matter) and the state slots shuffled."""
    from dli_amd.ops import seqmix
    torch.manual_seed(3)
    cols = Dv + int(normaliser)
    state_g = None
    starts = [0, 7, 0, 0, 0]
    for lens in ([1, 1, 2, 65, 190], [1, 64, 1, 3, 129]):
        mc, T = _step(lens, starts, "cpu")
        mg, _ = _step(lens, starts, "cuda")
        slots = int(max(mc.state_slots)) + 1
        if state_g is None:
            state_c = torch.randn(slots, H, D * cols) * 0.3
            state_g = state_c.cuda()
        q, k, v = torch.randn(T, G * D), torch.randn(T, G * D), torch.randn(T, H * Dv)
        if delta:
            q, k = (torch.nn.functional.normalize(x.view(T, G, D), dim=-1).view(T, G * D) for x in (q, k))
        q, k, v = (x.to(dtype) for x in (q, k, v))
        decay = -torch.exp(torch.empty(T, H).uniform_(-9.0, 3.0))
        weight = torch.rand(T, H)
        args = (mc, H, G, D, Dv, delta, 0.3, normaliser)
        want, wnq = seqmix.gated_scan(q, k, v, decay, weight, state_c, *args)
        got, gnq = seqmix.gated_scan(q.cuda(), k.cuda(), v.cuda(), decay.cuda(), weight.cuda(), state_g, mg, *args[1:])
        scale = float(want.abs().max())
        assert float((got.cpu() - want).abs().max()) < 2e-5 * max(scale, 1.0) * (1 if D < 200 else 2)
        if normaliser:
            assert float((gnq.cpu() - wnq).abs().max()) < 2e-5 * max(float(wnq.abs().max()), 1.0)
        assert float((state_g.cpu() - state_c).abs().max()) < 2e-5 * max(float(state_c.abs().max()), 1.0)
        starts = [s + n for s, n in zip(starts, lens)]


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_max_gates_against_the_reference(dtype):
    from dli_amd.ops import seqmix
    torch.manual_seed(5)
    H, lens, starts = 5, [1, 1300, 2, 513], [4, 0, 9, 0]
    mc, T = _step(lens, starts, "cpu")
    mg, _ = _step(lens, starts, "cuda")
    g = (torch.randn(T, 2 * H + 3) * 6).to(dtype)
    bias = torch.randn(2 * H)
    st_c = torch.randn(int(max(mc.state_slots)) + 1, H).abs()
    st_g = st_c.cuda()
    want = seqmix.max_gates(g, bias, 9.0, st_c, mc)
    got = seqmix.max_gates(g.cuda(), bias.cuda(), 9.0, st_g, mg)
    for a, b, name in zip(got, want, ("decay", "weight", "floor")):
        assert torch.allclose(a.cpu(), b, rtol=2e-5, atol=2e-5), name
    assert torch.allclose(st_g.cpu(), st_c, atol=2e-5)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("W", [256, 90])
def test_norm_and_gate_kernels_against_the_reference(W, dtype):
    from dli_amd.ops import seqmix
    torch.manual_seed(6)
    T = 37
    x = torch.randn(T, W)
    y, l, r = (torch.randn(T, W).to(dtype) for _ in range(3))
    wl, wr, w, b = (torch.randn(W) for _ in range(4))
    al = torch.tensor([0.8])
    cu = lambda t: t.cuda() if isinstance(t, torch.Tensor) else t
    tol = dict(rtol=1e-5, atol=1e-5) if dtype == torch.float32 else dict(rtol=1e-2, atol=1e-2)
    for yy, pair in ((None, None), (y, None), (y, (l, r, wl, wr)), (None, (l, r, wl, wr))):
        xc, xg = x.clone(), x.cuda()
        want = seqmix.residual_tanh_norm(xc, yy, pair, 0.4, al, w, b, 1e-4, dtype)
        got = seqmix.residual_tanh_norm(xg, cu(yy), tuple(cu(t) for t in pair) if pair else None, 0.4, al.cuda(), w.cuda(), b.cuda(), 1e-4, dtype)
        assert torch.allclose(xg.cpu(), xc, rtol=1e-5, atol=1e-5) and torch.allclose(got.cpu().float(), want.float(), **tol)
    wide = torch.randn(T, 2 * W + 8).to(dtype)
    buf = torch.zeros(T, W + 16, dtype=dtype)
    gbuf = buf.cuda()
    seqmix.gelu_rows(wide[:, 8:8 + W], out=buf[:, 16:])
    seqmix.gelu_rows(wide.cuda()[:, 8:8 + W], out=gbuf[:, 16:])
    assert torch.allclose(gbuf.cpu().float(), buf.float(), **tol) and float(gbuf[:, :16].abs().max()) == 0.0
    o, gate = torch.randn(T, W), torch.randn(T, W + 8).to(dtype)
    seq = torch.zeros(T, dtype=torch.int32)
    seq[-2:] = -1
    for groups in (1, 2):
        nq, fl, sk, c = torch.randn(T, 2), torch.rand(T, 2) + 0.1, torch.randn(T, W + 4), torch.randn(W // 2)
        for kw in (dict(divide=(nq, fl)), dict(skip=(sk[:, :W], c), gate_first=True), dict(gate_act="silu")):
            for wt in (torch.randn(W // groups), torch.randn(W)):
                want = seqmix.rms_gate(o, wt, 1e-4, gate[:, :W], dtype, groups=groups, **kw)
                kg = {k: tuple(t.cuda() for t in v) if isinstance(v, tuple) else v for k, v in kw.items()}
                if "skip" in kg:
                    kg["skip"] = (sk.cuda()[:, :W], c.cuda())
                out = torch.full((T, W + 24), 3.0, dtype=dtype, device="cuda")
                seqmix.rms_gate(o.cuda(), wt.cuda(), 1e-4, gate.cuda()[:, :W], dtype, groups=groups, out=out[:, 8:8 + W],
                                token_seq=seq.cuda(), **kg)
                assert torch.allclose(out[:-2, 8:8 + W].cpu().float(), want[:-2].float(), **tol)
                assert float(out[-2:, 8:8 + W].abs().max()) == 0.0 and float((out[:, :8] - 3).abs().max()) == 0.0
