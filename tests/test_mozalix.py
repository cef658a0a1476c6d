"""Mozalix stacks on the CPU path of the ops (fp32 torch references behind the same model, runner, block manager and
engine code as on the GPU) against the plain oracle ``mozalix_oracle``; plus the configuration reader, the loader and single
ops against the oracle's functions.  The GPU kernels run the same cases in ``test_mozalix_gpu.py``."""
import copy
import json
import os
import types

import pytest
import torch

import mozalix_cases as cases
import mozalix_oracle as oracle


@pytest.mark.parametrize("kind", sorted(cases.MECHANISMS))
def test_each_mechanism_alone(tmp_path, kind):
    cases.case_mechanism(tmp_path, "cpu", "float32", kind)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_every_piece_shows_when_wrong(tmp_path, dtype):
    cases.case_each_piece_matters(tmp_path, "cpu", dtype)


def test_prefill_decode_and_portions(tmp_path):
    cases.case_prefill_decode_portions(tmp_path, "cpu", "float32")


def test_unequal_requests_in_one_batch(tmp_path):
    cases.case_mixed_batch(tmp_path, "cpu", "float32")


def test_chunks_beside_single_tokens_at_matrix_core_sizes(tmp_path):
    cases.case_mixed_batch_on_tiles(tmp_path, "cpu", "float32")


def test_pages_and_slots_used_again(tmp_path):
    cases.case_reuse(tmp_path, "cpu", "float32")


def test_far_tokens(tmp_path):
    cases.case_far_token(tmp_path, "cpu", "float32")


@pytest.mark.parametrize("kind,place", cases.EDGES)
def test_keys_at_edges(tmp_path, kind, place):
    cases.case_edge(tmp_path, "cpu", "float32", kind, place)


def test_first_tokens_and_long_decoding(tmp_path):
    cases.case_first_tokens_and_long_decode(tmp_path, "cpu", "float32")


@pytest.mark.parametrize("name", sorted(cases.other_size_configs()))
def test_other_sizes(tmp_path, name):
    cases.case_other_sizes(tmp_path, "cpu", "float32", name)


def test_greedy_generation_through_the_engine(tmp_path):
    cases.case_generate(tmp_path, "cpu", "float32")


def test_layer_outputs_against_the_oracle(tmp_path):
    """The stream after every layer run, not only the logits."""
    from dli_amd.engine.trace import TraceReplayer
    W = cases.write_checkpoint(tmp_path, cases.FULL, 23)
    toks = cases.tokens(40, cases.FULL["vocab"], 9)
    want = oracle.forward(cases.resolved(cases.FULL), W, toks)[1]
    rep = TraceReplayer(str(tmp_path), "float32", 64, 2, "cpu")
    rep.runner.model.layer_outputs = got = []
    rep.step([{"id": "a", "tokens": toks, "want": []}], ["a"])
    assert len(got) == len(cases.FULL["layers"])
    for i, (g, w) in enumerate(zip(got, want)):
        assert torch.allclose(g.double(), w, rtol=2e-4, atol=2e-4 * float(w.abs().max())), f"after layer {i}"


def _load(cfg, path):
    """Configuration of a folder that holds ``cfg`` and its random weights."""
    from dli_amd.config import load_model_config
    cases.write_checkpoint(path, cfg, 0)
    return load_model_config(str(path), "float32")


def test_config_reader(tmp_path):
    from dli_amd.config import get_model_config, load_model_config, mozalix_config, resolve_model
    cases.write_checkpoint(tmp_path, cases.FULL, 1)
    cfg, path = resolve_model(str(tmp_path), "float32")
    assert path == str(tmp_path) and cfg.arch == "mozalix" and cfg.stateful and len(cfg.layer_specs) == 8
    assert (cfg.vocab_size, cfg.hidden_size, cfg.embed_scale, cfg.rms_eps, cfg.tie_embeddings) == (151, 72, 0.8, 1e-5, False)
    d, c, p = cfg.layer_specs[:3]
    assert (d.kind, d.heads, d.kv_heads, d.dim, d.vdim, d.window, d.chunk, d.maps, d.map_diff, d.rot_dims, d.rot_base, d.qk_weight, d.sink) == \
        ("masked_attention", 4, 2, 12, 20, 19, 0, 2, 0.3, 12, 700.0, True, False)
    assert (c.kind, c.heads, c.window, c.chunk, c.maps, c.rot_dims, c.scale, c.sink, c.score_cap) == ("masked_attention", 6, 0, 37, 1, 8, 0.3, True, 0.0)
    assert (c.ff, c.ff_act, c.ff_limit, c.ff_bias) == (92, "clamped", 1.6, True) and cfg.layer_specs[4].ff == 0
    a, b = p.parts
    assert (p.kind, p.part_scales, a.window, a.keep_first, a.score_cap, a.rot_dims, a.qk_weight, a.sink) == ("scaled_pair", (0.5, 1.2), 11, 2, 3.0, 0, False, False)
    assert (b.kind, b.heads, b.kv_heads, b.dim, b.vdim, b.conv_taps, b.lora, b.gate_lora) == ("channel_delta", 6, 2, 12, 20, 3, 6, 10)
    assert [s.weights_of for s in cfg.layer_specs] == [-1, -1, -1, 1, -1, 2, 0, 1]
    assert d.cache_row == (48, 40) and p.cache_row == (16, 28) and p.stateful and not d.stateful and p.state_shape == (6, 12, 20)
    assert get_model_config("tiny-mozalix").layer_specs[3].weights_of == 0
    broken = [cases.chunk(heads=5), cases.chunk(dims=7), cases.chunk(dims=40), cases.chunk(size=0), cases.diff(heads=3), cases.pair(cases.capped(cap=0.0)),
              cases.pair(right=cases.delta(heads=5)), cases.pair(right=cases.delta(conv=0)), cases.chunk(mlp={"kind": "moe", "ff": 8, "limit": 1.0}),
              cases.chunk(mlp={"kind": "dense", "ff": 8, "limit": 0.0}), {"type": "other", "mixer": {}, "mlp": None}]
    shapes = {"l0.mix.right.a1": (4, 72), "l0.mix.right.g1": (4, 72)}
    for bad in broken:
        with pytest.raises(ValueError):
            mozalix_config(cases.make_cfg([bad]), shapes=shapes)
    with pytest.raises(ValueError):                            # ranks from nowhere
        mozalix_config(cases.make_cfg([cases.pair()]))
    for wrong in (0, 2, 7, -1):                                # its own weights, nobody's, of a layer that differs
        cfg2 = cases.make_cfg([cases.chunk(), cases.diff()])
        cfg2["layers"][0]["weights_of" if wrong == 0 else "x"] = 0
        cfg2["layers"][1]["weights_of"] = wrong if wrong else 0
        with pytest.raises(ValueError):
            mozalix_config(cfg2)
    # the weights may belong to a layer that comes later
    later = cases.make_cfg([cases.chunk(), cases.chunk()])
    later["layers"][0]["weights_of"] = 1
    assert [s.weights_of for s in mozalix_config(later).layer_specs] == [1, -1]
    os.remove(tmp_path / "model.safetensors")
    with pytest.raises(ValueError):
        load_model_config(str(tmp_path))


def test_weights_of_a_later_layer(tmp_path):
    cfg = cases.make_cfg([cases.pair(mlp=cases.DENSE), cases.chunk(), cases.pair(mlp=cases.DENSE)])
    cfg["layers"][0]["weights_of"] = 2
    W, rig = cases._setup(tmp_path, cfg, "float32", "cpu", seed=8)
    toks = cases.tokens(60, cfg["vocab"], 3)
    cases._check(rig.run({"a": toks}, cases.alone("a", 60, [41, 1, 2, 16]))["a"], cases.expect(cfg, W, toks), "float32")


def test_fused_projections_state_sizes_and_parameter_count(tmp_path):
    from dli_amd.config import load_model_config
    from dli_amd.models import build_model
    W = cases.write_checkpoint(tmp_path, cases.FULL, 2)
    cfg = load_model_config(str(tmp_path), "float32")
    m = build_model(cfg, weights_path=str(tmp_path))
    assert cfg.param_count() == sum(t.numel() for t in W.values())
    assert sorted(m.layers) == ["0", "1", "2", "4"] and m.runs == ("0", "1", "2", "1", "4", "2", "0", "1")
    p = m.layers["2"]
    rows = torch.cat([W[f"l2.mix.left.{c}"] for c in "qkv"] + [W[f"l2.mix.right.{c}"] for c in ("q", "k", "v", "a1", "g1", "b")])
    assert torch.equal(p.inp.data[:rows.shape[0]], rows) and float(p.inp.data[rows.shape[0]:].abs().sum()) == 0.0
    assert p.inp.data.shape[0] % p.ALIGN == 0
    assert torch.equal(p.out.data, torch.cat([W["l2.mix.left.o"], W["l2.mix.right.o"]], dim=1))
    assert torch.equal(p.mixer.right.low.data, torch.block_diag(W["l2.mix.right.a2"], W["l2.mix.right.g2"]))
    assert torch.equal(m.layers["0"].mixer.lam.data, torch.stack([W[f"l0.mix.{c}"] for c in ("lq1", "lk1", "lq2", "lk2")]))
    one = 4 * (6 * 12 * 20 + 2 * (2 * 24 + 120))
    assert m.bytes_per_slot() == 2 * one + 4 * (4 * 16 * 8 + 4 * (2 * 64 + 32))
    assert m.bytes_per_block() == 32 * 4 * (2 * (48 + 40) + 3 * (40 + 24) + 2 * (16 + 28) + (24 + 32))
    c = m.allocate_caches(3, 2, "cpu")
    assert len(c) == 8 and c[1].k.shape == (3, 32, 40) and c[0].k.shape == (3, 32, 48) and c[2].parts[1].state.shape == (2, 6, 12, 20)
    assert c[1].k.data_ptr() != c[3].k.data_ptr()             # shared weights, caches of their own
    # random initialisation keeps the low-rank block structure and is reproducible
    r = build_model(cfg)
    low = r.layers["2"].mixer.right.low.data
    assert float(low[:72, 6:].abs().max()) == 0.0 == float(low[72:, :6].abs().max()) and float(low[:72, :6].std()) > 0.2
    assert torch.equal(low, build_model(cfg).layers["2"].mixer.right.low.data)


def _one_chunk(n, pos0=0, slot0=0):
    """Step metadata of one sequence bringing ``n`` tokens from position ``pos0`` (what the CPU references read)."""
    pos = torch.arange(pos0, pos0 + n, dtype=torch.int32)
    return types.SimpleNamespace(num_decode=0, num_prefill=1, query_start_loc=torch.tensor([0, n], dtype=torch.int32), slot_mapping=pos,
                                 state_slots=torch.tensor([0], dtype=torch.int32), positions=pos, block_tables=torch.arange(8, dtype=torch.int32)[None])


def test_small_ops_against_the_oracle():
    from dli_amd.ops import seqmix
    torch.manual_seed(1)
    # residual update with the norm behind a sublayer, with and without the closing norm
    x, y, w, w2 = torch.randn(5, 12), torch.randn(5, 12) * 1e-2, torch.randn(12), torch.randn(12)
    want = x.double() + oracle.stream_norm(y.double(), w.double(), 1e-3)
    a, b = x.clone(), x.clone()
    assert torch.allclose(seqmix.post_norm_add(a, y, w, 1e-3, torch.float32).double(), want, atol=1e-6) and torch.allclose(a.double(), want, atol=1e-6)
    assert torch.allclose(seqmix.post_norm_add(b, y, w, 1e-3, torch.float32, w2).double(), oracle.stream_norm(want, w2.double(), 1e-3), atol=1e-5)
    assert torch.allclose(b.double(), want, atol=1e-6)
    # embedding rows
    table = torch.randn(7, 12)
    ex, eh = seqmix.embed_rows(torch.tensor([3, 0, 6], dtype=torch.int32), table, 1.7, torch.bfloat16)
    assert torch.allclose(ex, table[[3, 0, 6]] * 1.7) and eh.dtype == torch.bfloat16
    # clamped activation: both sides of both bounds
    gu = torch.randn(6, 20) * 4
    want = oracle.feed_forward({"gate": torch.eye(20)[:10].double(), "up": torch.eye(20)[10:].double(), "down": torch.eye(10).double(),
                                "gate.b": 0.0, "up.b": 0.0, "down.b": 0.0}, "", {"limit": 2.0}, gu.double())
    assert torch.allclose(seqmix.act_mul(gu, "clamped", 2.0).double(), want, atol=1e-5)
    # convolution with write strengths instead of step gates
    cx, cw, g = torch.randn(9, 10), torch.randn(10, 4), torch.randn(9, 3)
    got, _, beta = seqmix.causal_conv(cx, cw.t().contiguous(), None, torch.full((1, 3, 10), 7.0), _one_chunk(9), torch.float32, act="silu",
                                      gates=("beta", g, torch.ones(3), torch.ones(3)))
    assert torch.allclose(got.double(), oracle.silu(oracle.causal_conv(cx.double(), cw.double())), atol=1e-5)
    assert torch.allclose(beta, torch.sigmoid(g))
    # two maps
    T, H, G, Dv = 4, 6, 2, 10
    a1, a2 = torch.randn(T, H, Dv), torch.randn(T, H, Dv)
    o = torch.stack([a1.view(T, G, 3, Dv), a2.view(T, G, 3, Dv)], dim=2).reshape(T, 2 * H, Dv)
    out = torch.zeros(T, H * Dv + 4)
    seqmix.map_combine(o, torch.tensor([0.3]), 1e-4, 0.8, G, out[:, 4:])
    assert torch.allclose(out[:, 4:].double(), (oracle.rms((a1 - 0.3 * a2).double(), 1e-4) * 0.8).reshape(T, -1), atol=1e-5)
    assert float(out[:, :4].abs().max()) == 0.0


@pytest.mark.parametrize("maps", [1, 2])
def test_head_norm_and_rotation_against_the_oracle(maps):
    from dli_amd.ops import seqmix
    torch.manual_seed(2)
    T, H, G, D, Dv, dims = 11, 6, 2, 10, 4, 6
    proj = torch.randn(T, (H + G) * maps * D + G * Dv + 3)[:, :-3]
    qw, kw = torch.rand(D) + 0.5, torch.rand(D) + 0.5
    rot = {"base": 900.0, "dims": dims}
    for weights in ((qw, kw), (None, None)):
        kc, vc = torch.zeros(1, 32, G * maps * D), torch.zeros(1, 32, G * Dv)
        q = seqmix.head_norm_rope_cache(proj, *weights, 1e-4, torch.arange(T, dtype=torch.int32), seqmix.rotary_inv_freq(900.0, dims), dims,
                                        torch.arange(T, dtype=torch.int32), kc, vc, H, G, D, Dv, maps)
        W = {"q.norm": qw.double(), "k.norm": kw.double()} if weights[0] is not None else {}
        nq, nk = H * maps * D, G * maps * D
        wq, wk = oracle.normed_qk(W, "", proj[:, :nq].double().view(T, H, maps, D), proj[:, nq:nq + nk].double().view(T, G, maps, D), rot, 1e-4)
        assert torch.allclose(kc[0, :T].double(), wk.reshape(T, -1), atol=1e-5) and torch.equal(vc[0, :T], proj[:, nq + nk:])
        for h in range(H):                                     # order: key head, map, head of its group
            for m in range(maps):
                i = (h // 3 * maps + m) * 3 + h % 3
                assert torch.allclose(q[:, i].double(), wq[:, h, m], atol=1e-5)


def test_masks_of_the_attention_reference_against_the_oracle():
    """Every mask over all positions of a sequence, in portions; scores that make single keys matter."""
    from dli_amd.ops import seqmix
    torch.manual_seed(3)
    T, H, G, D, Dv = 80, 4, 2, 8, 6
    q, k, v = torch.randn(T, H, D) * 2, torch.randn(T, G, D) * 2, torch.randn(T, G, Dv)
    sink = torch.randn(H)
    kc, vc = torch.zeros(8, 32, G * D), torch.zeros(8, 32, G * Dv)
    kc.view(-1, G * D)[:T], vc.view(-1, G * Dv)[:T] = k.reshape(T, -1), v.reshape(T, -1)
    qd, kd, vd = (t.double() for t in (q, k, v))
    for kw, see, cap, sk in ((dict(chunk=13), oracle.visible(T, "chunk", {"size": 13}), None, sink), (dict(window=9), oracle.visible(T, "window", {"size": 9}), None, None),
                             (dict(window=9, keep_first=4, cap=2.0), oracle.visible(T, "keep", {"size": 9, "keep_first": 4}), 2.0, None),
                             (dict(window=1, keep_first=40, cap=2.0), oracle.visible(T, "keep", {"size": 1, "keep_first": 40}), 2.0, None)):
        out = torch.zeros(T, H, Dv)
        for a, b in ((0, 33), (33, 34), (34, 80)):
            seqmix.token_attention(out[a:b], q[a:b], None, kc, vc, _one_chunk(b - a, a), G, Dv, 0.5, sink=sk, out_scale=0.7, **kw)
        want = 0.7 * oracle.softmax_attention(qd, kd, vd, 0.5, see, cap, sk.double() if sk is not None else None)
        assert torch.allclose(out.double(), want, atol=1e-5), kw


def test_channel_decays_against_the_oracle():
    from dli_amd.ops import seqmix
    torch.manual_seed(4)
    T, H, G, D, Dv = 30, 4, 2, 6, 5
    q, k, v = torch.randn(T, G * D), torch.nn.functional.normalize(torch.randn(T, G, D), dim=-1).view(T, G * D), torch.randn(T, H * Dv)
    z, rate, bias, beta = torch.randn(T, H * D) * 2, torch.rand(H) + 0.1, torch.randn(H * D), torch.rand(T, H)
    st = torch.full((1, H, D, Dv), 5.0)
    got = torch.cat([seqmix.channel_delta_scan(q[a:b], k[a:b], v[a:b], z[a:b], rate, bias, beta[a:b], st, _one_chunk(b - a, a), H, G, D, Dv)
                     for a, b in ((0, 7), (7, 8), (8, 30))])
    g = torch.exp(-rate.double()[:, None] * oracle.softplus((z + bias).double()).view(T, H, D))
    rep = lambda t: t.double().view(T, G, D).repeat_interleave(H // G, dim=1)
    want = oracle.channel_delta_scan(rep(q), rep(k), v.double().view(T, H, Dv), g, beta.double())
    assert torch.allclose(got.double().view(T, H, Dv), want, atol=1e-5)


def test_oracle_follows_weights_of(tmp_path):
    """A layer on another's weights equals a copy of them."""
    W = cases.write_checkpoint(tmp_path, cases.FULL, 6)
    toks = cases.tokens(20, cases.FULL["vocab"], 1)
    plain = copy.deepcopy(cases.resolved(cases.FULL))
    W2 = dict(W)
    for i, L in enumerate(plain["layers"]):
        src = L.pop("weights_of", None)
        if src is not None:
            W2.update({f"l{i}." + k.split(".", 1)[1]: v for k, v in W.items() if k.startswith(f"l{src}.")})
    assert cases.rel_err(oracle.forward(plain, W2, toks)[0].numpy(), cases.expect(cases.FULL, W, toks)) == 0.0
    assert json.dumps(cases.FULL)                              # the case configuration itself stays as it was
