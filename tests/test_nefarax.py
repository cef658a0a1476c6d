"""Nefarax stacks on the CPU path of the ops (fp32 torch references behind the same model, runner, block manager and
engine code as on the GPU) against the plain oracle ``nefarax_oracle``; plus the configuration reader, the loader and single
ops against the oracle's functions.  The GPU kernels run the same cases in ``test_nefarax_gpu.py``."""
import json
import os
import types

import pytest
import torch

import nefarax_cases as cases
import nefarax_oracle as oracle


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


@pytest.mark.parametrize("which", sorted(cases.FAR))
def test_far_tokens(tmp_path, which):
    cases.case_far_token(tmp_path, "cpu", "float32", which)


@pytest.mark.parametrize("place", [31, 32, 63])
def test_keys_at_page_borders(tmp_path, place):
    cases.case_page_border(tmp_path, "cpu", "float32", place)


def test_first_tokens_and_long_decoding(tmp_path):
    cases.case_first_tokens_and_long_decode(tmp_path, "cpu", "float32")


@pytest.mark.parametrize("name", sorted(cases.other_size_configs()))
def test_other_sizes(tmp_path, name):
    cases.case_other_sizes(tmp_path, "cpu", "float32", name)


def test_greedy_generation_through_the_engine(tmp_path):
    cases.case_generate(tmp_path, "cpu", "float32")


def test_layer_outputs_against_the_oracle(tmp_path):
    """The stream after every layer, not only the logits."""
    from dli_amd.engine.trace import TraceReplayer
    W = cases.write_checkpoint(tmp_path, cases.FULL, 23)
    toks = cases.tokens(40, cases.FULL["vocab"], 9)
    want = oracle.forward(cases.FULL, W, toks)[1]
    rep = TraceReplayer(str(tmp_path), "float32", 64, 2, "cpu")
    rep.runner.model.layer_outputs = got = []
    rep.step([{"id": "a", "tokens": toks, "want": []}], ["a"])
    assert len(got) == len(cases.FULL["layers"])
    for i, (g, w) in enumerate(zip(got, want)):
        assert torch.allclose(g.double(), w, rtol=2e-4, atol=2e-4 * float(w.abs().max())), f"after layer {i}"


def _load(cfg, path):
    from dli_amd.config import load_model_config
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as fh:
        json.dump(cfg, fh)
    return load_model_config(str(path), "float32")


def test_config_reader(tmp_path):
    from dli_amd.config import get_model_config, resolve_model
    cases.write_checkpoint(tmp_path, cases.FULL, 1)
    cfg, path = resolve_model(str(tmp_path), "float32")
    assert path == str(tmp_path) and cfg.arch == "nefarax" and cfg.stateful and cfg.tie_embeddings and len(cfg.layer_specs) == 6
    assert (cfg.vocab_size, cfg.hidden_size, cfg.residual_mult, cfg.rms_eps) == (149, 72, 0.6, 1e-5)
    m, d, p = cfg.layer_specs[:3]
    assert (m.kind, m.heads, m.dim, m.vdim, m.gate_cap, m.ff, m.ff_act) == ("mlstm", 3, 16, 24, 4.0, 88, "gelu_tanh_plain")
    assert (d.kind, d.heads, d.kv_heads, d.dim, d.vdim, d.conv_taps) == ("delta", 6, 2, 12, 20, 3)
    a, s = p.parts
    assert (p.kind, a.kind, s.kind) == ("normed_pair", "conv_attention", "ssd")
    assert (a.heads, a.kv_heads, a.dim, a.conv_taps, a.scale, a.rot_dims, a.rot_base, a.rot_scaling) == (6, 3, 20, 4, 0.3, 12, 3000.0, (4.0, 96.0, 8.0, 2.0))
    assert (s.heads, s.vdim, s.dim, s.kv_heads, s.conv_taps, s.norm_groups) == (6, 12, 20, 3, 3, 4)
    assert p.cache_row == (60, 60) and d.cache_row == (0, 0) and p.stateful and cfg.layer_specs[3].ff == 0
    assert get_model_config("tiny-nefarax").arch == "nefarax"
    plain = _load(cases.make_cfg([cases.pair(cases.attn(dims=0))]), tmp_path / "plain").layer_specs[0].parts[0]
    assert plain.rot_dims == 0 and plain.rot_scaling == ()
    wrong_values = cases.attn()
    wrong_values["vdim"] = 8
    for bad in (cases.delta(heads=5), cases.delta(conv=0), cases.pair(cases.attn(heads=4)), cases.pair(cases.attn(dims=7)),
                cases.pair(cases.attn(dims=40)), cases.pair(wrong_values), cases.pair(right=cases.ssd(groups=4)),
                cases.pair(right=cases.ssd(norm_groups=5)), cases.mlstm(gate_cap=0.0), cases.delta(mlp={"kind": "moe", "ff": 8}),
                {"type": "other", "mixer": {}, "mlp": None}):
        with pytest.raises(ValueError):
            _load(cases.make_cfg([bad]), tmp_path / "bad")


def test_fused_projections_state_sizes_and_parameter_count(tmp_path):
    from dli_amd.config import load_model_config
    from dli_amd.models import build_model
    W = cases.write_checkpoint(tmp_path, cases.FULL, 2)
    cfg = load_model_config(str(tmp_path), "float32")
    m = build_model(cfg, weights_path=str(tmp_path))
    assert cfg.param_count() == sum(t.numel() for t in W.values())
    d = m.layers[1]                                            # delta rule with a feed-forward
    rows = torch.cat([W["l1.mlp.up"]] + [W[f"l1.mix.{c}"] for c in "qkvgba"])
    assert torch.equal(d.inp.data[:rows.shape[0]], rows) and float(d.inp.data[rows.shape[0]:].abs().sum()) == 0.0
    assert d.inp.data.shape[0] % d.ALIGN == 0
    assert torch.equal(d.out.data, torch.cat([W["l1.mix.o"], W["l1.mlp.down"]], dim=1))
    assert m.layers[4].out is None and torch.equal(m.layers[2].out.data, W["l2.mlp.down"])
    per_slot = sum(4 * n for n in (3 * 16 * 25 + 3,            # mlstm: state and normaliser, running maximum
                                   6 * 12 * 20 + 2 * (48 + 120), 4 * 16 * 8 + 4 * (128 + 32),
                                   6 * 20 * 12 + 2 * (72 + 120) + 3 * 180, 4 * 16 * 10 + 4 * (40 + 32) + 80, 2 * 24 * 17 + 2))
    assert m.bytes_per_slot() == per_slot
    assert m.bytes_per_block() == 32 * 4 * (2 * 60 + 2 * 16)
    c = m.allocate_caches(3, 2, "cpu")
    assert len(c[2].state_tensors()) == 3 and len(c[0].state_tensors()) == 2 and c[2].parts[0].k.shape == (3, 32, 60)
    assert build_model(load_model_config_like(cfg)).bytes_per_block() >= 1


def load_model_config_like(cfg):
    """The same configuration without its attention layers: no paged rows at all."""
    import dataclasses
    return dataclasses.replace(cfg, layer_specs=tuple(s for s in cfg.layer_specs if s.kind != "normed_pair"))


def _one_chunk(n, pos0=0):
    """Step metadata of one sequence bringing ``n`` tokens from position ``pos0`` (what the CPU references read)."""
    return types.SimpleNamespace(num_decode=0, num_prefill=1, query_start_loc=torch.tensor([0, n], dtype=torch.int32),
                                 state_slots=torch.tensor([0], dtype=torch.int32), positions=torch.arange(pos0, pos0 + n, dtype=torch.int32))


def test_frequency_bands_against_the_oracle():
    from dli_amd.ops import seqmix
    for sc in ({"factor": 4.0, "high": 8.0, "low": 2.0, "original": 96}, {"factor": 32.0, "high": 4.0, "low": 1.0, "original": 8192}, None):
        rot = {"base": 20000.0, "dims": 40, "scaling": sc}
        f = seqmix.banded_inv_freq(20000.0, 40, (sc["factor"], sc["original"], sc["high"], sc["low"]) if sc else ())
        want = torch.tensor(oracle.frequencies(rot), dtype=torch.float64)
        assert torch.allclose(f, want, rtol=1e-12)
        if sc:                                                 # all three bands occur
            plain = torch.tensor(oracle.frequencies(rot, plain=True), dtype=torch.float64)
            ratio = want / plain
            assert (ratio == 1).any() and (ratio < 1.0001 / sc["factor"]).any() and ((ratio < 0.99) & (ratio > 1.01 / sc["factor"])).any()


def test_small_ops_against_the_oracle():
    from dli_amd.ops import seqmix
    torch.manual_seed(1)
    # convolution with silu, unit vectors and gates; in two portions through the state rows of a reused slot
    x, w = torch.randn(9, 10), torch.randn(10, 4)
    g, rate, bias = torch.randn(9, 6), torch.rand(3) + 0.2, torch.randn(3)
    y = oracle.silu(oracle.causal_conv(x.double(), w.double()))
    want = torch.cat([oracle.unit(y[:, :3]) * 0.5, oracle.unit(y[:, 3:6]), y[:, 6:]], dim=1)
    st = torch.full((1, 3, 10), 7.0)
    parts = [seqmix.causal_conv(x[a:b], w.t().contiguous(), None, st, _one_chunk(b - a, a), torch.float32, act="silu", unit=(2, 3, 1, 0.5),
                                gates=("delta", g[a:b], rate, bias)) for a, b in ((0, 2), (2, 9))]
    got, la, wt = (torch.cat(t) for t in zip(*parts))
    assert torch.allclose(got.double(), want, atol=1e-5)
    assert torch.allclose(la.double(), -rate.double() * oracle.softplus(g[:, 3:].double() + bias.double()), atol=1e-5)
    assert torch.allclose(wt, torch.sigmoid(g[:, :3]))
    # gates with a running maximum, in two portions
    gg, b2 = torch.randn(11, 4) * 5, torch.randn(4)
    st = torch.full((1, 2), 9.0)
    parts = [seqmix.max_gates(gg[a:b], b2, 3.0, st, _one_chunk(b - a, a)) for a, b in ((0, 4), (4, 11))]
    keep, write, floor = (torch.cat(t) for t in zip(*parts))
    z = 3.0 * torch.tanh((gg + b2).double() / 3.0)
    m = torch.zeros(2, dtype=torch.float64)
    for t in range(11):
        f = oracle.logsigmoid(z[t, 2:])
        new = torch.maximum(f + m, z[t, :2])
        for a, b in ((keep[t], f + m - new), (write[t], torch.exp(z[t, :2] - new)), (floor[t], torch.exp(-new))):
            assert torch.allclose(a.double(), b, atol=1e-5)
        m = new
    # residual update with a pair, and the norm
    xs, yv, l, r, wl, wr, wn, bn = (torch.randn(*s) for s in ((5, 12), (5, 12), (5, 12), (5, 12), (12,), (12,), (12,), (12,)))
    al = torch.tensor([0.7])
    want = xs.double() + 0.3 * (yv + 0.5 * (oracle.rms(l.double(), 1e-3) * wl + oracle.rms(r.double(), 1e-3) * wr))
    got = seqmix.residual_tanh_norm(xs, yv, (l, r, wl, wr), 0.3, al, wn, bn, 1e-3, torch.float32)
    assert torch.allclose(xs.double(), want, atol=1e-5)
    assert torch.allclose(got.double(), oracle.tanh_norm(want, 0.7, wn.double(), bn.double()), atol=1e-5)
    # norm and gate behind a recurrence: divisor, shared weight; skip term and leading gate
    o, gate, nq, fl = torch.randn(4, 12), torch.randn(4, 12), torch.randn(4, 3), torch.rand(4, 3)
    w4 = torch.randn(4)
    den = torch.maximum(nq.abs(), fl).double() + 1e-6
    want = (oracle.rms(o.double().view(4, 3, 4) / den[:, :, None], 1e-5) * w4).reshape(4, 12) * torch.sigmoid(gate.double())
    assert torch.allclose(seqmix.rms_gate(o, w4, 1e-5, gate, torch.float32, groups=3, divide=(nq, fl)).double(), want, atol=1e-5)
    sk, c, w12 = torch.randn(4, 12), torch.randn(6), torch.randn(12)
    v = (o.double() + (sk.view(4, 6, 2) * c.view(1, 6, 1)).reshape(4, 12)) * oracle.silu(gate.double())
    want = oracle.rms(v.view(4, 2, 6), 1e-5).reshape(4, 12) * w12
    assert torch.allclose(seqmix.rms_gate(o, w12, 1e-5, gate, torch.float32, groups=2, gate_act="silu", skip=(sk, c), gate_first=True).double(), want,
                          atol=1e-5)
