"""Prefill and decode throughput of Rodelix stacks at layer sizes of a real model, beside a Llama stack of equal
size (same width, heads, head size and parameter count per layer), both with random weights, both through the same
engine: requests are added to ``LLMEngine`` and stepped by its scheduler; prefill is timed with one-token requests
(prompt tokens / wall time), decoding from the step in which the last request got its first token to the end.

    python bench.py --mixers                     # all sizes, one JSON line per (size, model)
    python benchmarks/bench_mixers.py --sizes small --prompt 1024 --batch 32

Sizes: ``small`` = width 2048, 16 heads of 128, 4 KV heads, FFN 8192 (Llama) — ``large`` = width 4096, 32 heads of 128,
8 KV heads, FFN 14336 (a Llama-3-8B layer).  The Rodelix stack has one layer per mixer (window attention of 1024 tokens,
lightning, latent attention with a 512-wide latent + 64 rotated) and a squared-ReLU FFN of 1.5× the Llama FFN width (two
matrices instead of three: equal parameters); ``rodelix-<mixer>`` rows repeat ONE mixer in every layer so that the three
can be told apart.  Vocabulary 32000 for all.

``--models mixtral,vibunex`` compares the gated parallel stack (sink attention beside a time-mix recurrence, routed
squared-ReLU experts) with the closest existing family, a Mixtral stack of the same width, heads and head size: 8 experts,
2 per token, Mixtral expert width = half the Llama FFN; the Vibunex experts are 1.5× as wide minus 512 with a shared expert
of 1024 (two matrices instead of three: the same feed-forward FLOPs per token); its recurrence has width / 64 heads of 64.

``--models mixtral,llama,rodelix-lightning,sevelorn,sevelorn-attention,sevelorn-retention`` compares the hyper-connected
stacks (four fp32 streams, a four-tap input convolution) with their closest families at equal width, heads and head size:
``sevelorn-attention`` = gated attention (every layer with keys / values of its own) + 8 silu experts, 2 per token, of the
Mixtral expert width — beside ``mixtral``; ``sevelorn-retention`` = retention (heads of 128 × 128) + a tanh-GELU gated
feed-forward of the Llama width — beside ``rodelix-lightning`` (mixer) and ``llama`` (feed-forward); ``sevelorn`` = an
attention layer, an attention layer on the first one's keys / values (both with experts) and a retention layer (dense).

``--models rodelix-lightning,sinilorn-recurrence,rodelix-latent_attention,sinilorn-latent,mixtral,sinilorn`` compares the
Sinilorn stacks (four fp32 streams read through a layer norm) with their closest families: ``sinilorn-recurrence`` = a gated
linear recurrence over ``width`` channels in blocks of 128 behind a four-tap convolution + a silu-gated dense feed-forward with
biases of the Llama width — beside ``rodelix-lightning`` (the framework's other recurrent mixer); ``sinilorn-latent`` = gated
latent attention (512-wide latent + 64 rotated, queries through a latent of 3/4 of the width, window 1024, sink, output gate)
+ 8 clamped experts and 2 identity experts, 2 per token, of the Mixtral expert width — beside ``rodelix-latent_attention``
(mixer) and ``mixtral`` (experts); ``sinilorn`` = a recurrence (dense), a latent layer and a latent layer on the second
one's cache rows (both with experts).

``--models rodelix-lightning,nefarax-delta,nefarax-mlstm,rodelix-attention,nefarax-pair,nefarax`` compares the Nefarax stacks (one
tanh norm per layer, mixer and plain tanh-GELU feed-forward of 1.5× the Llama FFN width side by side) with their closest families:
``nefarax-delta`` = the gated delta rule (half as many q / k heads as value heads, heads of 128 × 128, four-tap convolutions) and
``nefarax-mlstm`` = mLSTM (heads of 128 × 128) — both beside ``rodelix-lightning``, the framework's other ``[128, 128]`` state per head;
``nefarax-pair`` = convolved attention beside a Mamba-2 recurrence (inner width twice the model width in heads of 64, state 128) —
beside ``rodelix-attention`` (attention) and ``rodelix-lightning`` (recurrence); ``nefarax`` = one layer of each.

``--models rodelix-attention,mozalix-chunk,mozalix-diff,nefarax-delta,mozalix-delta,mozalix-pair,llama,mozalix`` compares the Mozalix
stacks (post-norm layers on the unnormed stream, a clamped gated feed-forward with biases of the Llama FFN width) with their closest
families: ``mozalix-chunk`` = attention in chunks of 1024 with a sink and ``mozalix-diff`` = differential attention over a window of 1024
(two maps of 64 per head of 128) — both beside ``rodelix-attention`` (window 1024); ``mozalix-pair`` = soft-capped window attention
(1024, four kept tokens) beside the delta rule with channel decays (half as many q / k heads as value heads, heads of 128 × 128,
four taps, both low ranks 128) — beside ``rodelix-attention`` and ``nefarax-delta``; ``mozalix-delta`` = the same with the attention half cut to
one head of 16 over a window of 32, for the recurrence alone; ``mozalix`` = one layer of chunk, diff and pair.
"""
from __future__ import annotations

import argparse
import json
import os
import sys
import time

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
if ROOT not in sys.path:
    sys.path.insert(0, ROOT)

SIZES = {"small": dict(width=2048, heads=16, kv=4, ffn=8192), "large": dict(width=4096, heads=32, kv=8, ffn=14336)}
LAYERS = 3


def rodelix_raw(width, heads, kv, ffn, mixers):
    ff = {"kind": "dense", "ff": ffn * 3 // 2}
    mk = {
        "attention": {"type": "attention", "mlp": ff, "mixer": {"heads": heads, "kv_heads": kv, "dim": 128, "vdim": 128,
                                                                  "scale": 128 ** -0.5, "mask": {"size": 1024}}},
        "lightning": {"type": "lightning", "mlp": ff, "mixer": {"heads": heads, "dim": 128, "vdim": 128,
                                                                  "decay": [1.0 - 2.0 ** -(3 + 5 * h / heads) for h in range(heads)]}},
        "latent_attention": {"type": "latent_attention", "mlp": ff,
                             "mixer": {"heads": heads, "dim": 128, "rot_dim": 64, "vdim": 128, "kv_rank": 512,
                                       "scale": 192 ** -0.5, "rot": {"base": 10000.0, "dims": 64}}},
    }
    return {"architecture": "Rodelix", "vocab": 32000, "width": width, "residual_mult": 0.5, "logit_softcap": 30.0,
            "norm": {"eps": 1e-5}, "layers": [mk[m] for m in mixers]}


def vibunex_raw(width, heads, kv, ffn):
    inner = ffn // 2
    layer = {"type": "parallel",
             "mixer": {"left_scale": 0.7, "right_scale": 0.7,
                       "left": {"heads": heads, "kv_heads": kv, "dim": 128, "vdim": 128, "scale": 128 ** -0.5,
                                "rot": {"base": 1000000.0, "dims": 64,
                                        "scaling": {"factor": 8.0, "original": 8192, "fast": 16.0, "slow": 2.0}}},
                       "right": {"heads": width // 64, "dim": 64, "lora": 64}},
             "mlp": {"kind": "moe", "expert": {"ff": inner * 3 // 2 - 512}, "router": {"experts": 8, "top": 2, "scale": 1.0},
                     "shared": {"ff": 1024}}}
    return {"architecture": "Vibunex", "vocab": 32000, "width": width, "residual_mult": 0.5, "norm": {"eps": 1e-5},
            "layers": [layer] * LAYERS}


def sevelorn_raw(width, heads, kv, ffn, kinds):
    moe = {"kind": "moe", "expert": {"ff": ffn // 2}, "router": {"experts": 8, "top": 2}}
    dense = {"kind": "dense", "ff": ffn}
    att = {"heads": heads, "kv_heads": kv, "dim": 128, "vdim": 128, "scale": 128 ** -0.5}
    mk = {
        "attention": {"type": "attention", "mlp": moe, "mixer": att},
        "shared_attention": {"type": "attention", "mlp": moe, "mixer": dict(att, kv_from=0)},
        "retention": {"type": "retention", "mlp": dense,
                      "mixer": {"heads": heads, "dim": 128, "vdim": 128, "rot": {"base": 1000000.0, "dims": 128},
                                "decay": [1.0 - 2.0 ** -(3 + 5 * h / heads) for h in range(heads)]}},
    }
    return {"architecture": "Sevelorn", "vocab": 32000, "width": width, "streams": 4, "canon": {"taps": 4},
            "embedding": {"scale": 1.0}, "norm": {"eps": 1e-5}, "layers": [mk[k] for k in kinds]}


def sinilorn_raw(width, heads, kv, ffn, kinds):
    moe = {"kind": "moe", "expert": {"ff": ffn // 2, "limit": 7.0}, "router": {"experts": 8, "identity": 2, "top": 2}}
    dense = {"kind": "dense", "ff": ffn}
    lat = {"heads": heads, "dim": 128, "rot_dim": 64, "vdim": 128, "kv_rank": 512, "q_rank": width * 3 // 4, "scale": 192 ** -0.5,
           "mask": {"size": 1024},
           "rot": {"base": 1000000.0, "dims": 64, "scaling": {"factor": 8.0, "original": 8192, "fast": 16.0, "slow": 2.0}}}
    mk = {
        "recurrence": {"type": "rglru", "mlp": dense, "mixer": {"blocks": width // 128, "conv": 4, "width": width}},
        "latent": {"type": "latent_attention", "mlp": moe, "mixer": lat},
        "shared_latent": {"type": "latent_attention", "mlp": moe, "mixer": dict(lat, kv_from=1)},
    }
    return {"architecture": "Sinilorn", "vocab": 32000, "width": width, "streams": 4, "logit_scale": 1.0, "norm": {"eps": 1e-5},
            "layers": [mk[k] for k in kinds]}


def nefarax_raw(width, heads, kv, ffn, kinds):
    ff = {"kind": "dense", "ff": ffn * 3 // 2}
    mk = {
        "delta": {"type": "delta", "mlp": ff, "mixer": {"heads": heads, "kv_heads": heads // 2, "dim": 128, "vdim": 128, "conv": 4}},
        "mlstm": {"type": "mlstm", "mlp": ff, "mixer": {"heads": heads, "dim": 128, "vdim": 128, "gate_cap": 12.0}},
        "pair": {"type": "parallel", "mlp": ff,
                 "mixer": {"left": {"heads": heads, "kv_heads": kv, "dim": 128, "vdim": 128, "conv": 4, "scale": 128 ** -0.5,
                                    "rot": {"base": 500000.0, "dims": 128, "scaling": {"factor": 8.0, "high": 4.0, "low": 1.0, "original": 8192}}},
                           "right": {"heads": 2 * width // 64, "vdim": 64, "state": 128, "groups": 1, "conv": 4, "norm_groups": 1}}},
    }
    return {"architecture": "Nefarax", "vocab": 32000, "width": width, "residual_mult": 0.5, "norm": {"eps": 1e-5},
            "layers": [mk[k] for k in kinds]}


def mozalix_raw(width, heads, kv, ffn, kinds):
    ff = {"kind": "dense", "ff": ffn, "limit": 7.0}
    att = {"heads": heads, "kv_heads": kv, "dim": 128, "vdim": 128, "scale": 128 ** -0.5, "mask": {"size": 1024}}
    left = dict(att, softcap=30.0, mask={"size": 1024, "keep_first": 4})
    little = {"heads": 1, "kv_heads": 1, "dim": 16, "vdim": 16, "scale": 0.25, "softcap": 30.0, "mask": {"size": 32, "keep_first": 0}}
    right = {"heads": heads, "kv_heads": heads // 2, "dim": 128, "vdim": 128, "conv": 4, "lora": 128, "gate_lora": 128}
    mk = {
        "chunk": {"type": "attention", "mlp": ff, "mixer": dict(att, rot={"base": 500000.0, "dims": 64})},
        "diff": {"type": "attention_2", "mlp": ff, "mixer": dict(att, dim=64, scale=0.125, diff=0.5, rot={"base": 500000.0, "dims": 64})},
        "pair": {"type": "parallel", "mlp": ff, "mixer": {"left_scale": 0.7, "right_scale": 0.7, "left": left, "right": right}},
        "delta": {"type": "parallel", "mlp": ff, "mixer": {"left_scale": 0.7, "right_scale": 0.7, "left": little, "right": right}},
    }
    return {"architecture": "Mozalix", "vocab": 32000, "width": width, "embedding": {"scale": 1.0}, "norm": {"eps": 1e-5},
            "layers": [mk[k] for k in kinds]}


def model_configs(size):
    from dli_amd.config import ModelConfig, mozalix_config, nefarax_config, rodelix_config, sevelorn_config, sinilorn_config, vibunex_config
    s = SIZES[size]
    out = {"llama": ModelConfig(name=f"llama-{size}", arch="llama", vocab_size=32000, hidden_size=s["width"],
                                intermediate_size=s["ffn"], num_layers=LAYERS, num_heads=s["heads"], num_kv_heads=s["kv"],
                                head_dim=128, max_position=16384)}
    out["mixtral"] = ModelConfig(name=f"mixtral-{size}", arch="mixtral", vocab_size=32000, hidden_size=s["width"],
                                 intermediate_size=s["ffn"] // 2, num_layers=LAYERS, num_heads=s["heads"], num_kv_heads=s["kv"],
                                 head_dim=128, max_position=16384, num_experts=8, top_k_experts=2)
    out["vibunex"] = vibunex_config(vibunex_raw(s["width"], s["heads"], s["kv"], s["ffn"]), name=f"vibunex-{size}")
    for name, kinds in (("sevelorn", ("attention", "shared_attention", "retention")), ("sevelorn-attention", ("attention",) * LAYERS),
                        ("sevelorn-retention", ("retention",) * LAYERS)):
        out[name] = sevelorn_config(sevelorn_raw(s["width"], s["heads"], s["kv"], s["ffn"], kinds), name=f"{name}-{size}")
    for name, kinds in (("sinilorn", ("recurrence", "latent", "shared_latent")), ("sinilorn-recurrence", ("recurrence",) * LAYERS),
                        ("sinilorn-latent", ("latent",) * LAYERS)):
        out[name] = sinilorn_config(sinilorn_raw(s["width"], s["heads"], s["kv"], s["ffn"], kinds), name=f"{name}-{size}")
    for name, kinds in (("nefarax", ("delta", "mlstm", "pair")), ("nefarax-delta", ("delta",) * LAYERS), ("nefarax-mlstm", ("mlstm",) * LAYERS),
                        ("nefarax-pair", ("pair",) * LAYERS)):
        out[name] = nefarax_config(nefarax_raw(s["width"], s["heads"], s["kv"], s["ffn"], kinds), name=f"{name}-{size}")
    for name, kinds in (("mozalix", ("chunk", "diff", "pair")), ("mozalix-chunk", ("chunk",) * LAYERS), ("mozalix-diff", ("diff",) * LAYERS),
                        ("mozalix-pair", ("pair",) * LAYERS), ("mozalix-delta", ("delta",) * LAYERS)):
        out[name] = mozalix_config(mozalix_raw(s["width"], s["heads"], s["kv"], s["ffn"], kinds), name=f"{name}-{size}")
    kinds = ("attention", "lightning", "latent_attention")
    out["rodelix"] = rodelix_config(rodelix_raw(s["width"], s["heads"], s["kv"], s["ffn"], kinds), name=f"rodelix-{size}")
    for k in kinds:
        out[f"rodelix-{k}"] = rodelix_config(rodelix_raw(s["width"], s["heads"], s["kv"], s["ffn"], (k,) * LAYERS),
                                             name=f"rodelix-{k}-{size}")
    return out


def run_one(mcfg, prompt, batch, new_tokens, device="cuda", graphs=True):
    import numpy as np
    import torch
    from dli_amd.config import CacheConfig, EngineConfig, SamplingParams, SchedulerConfig
    from dli_amd.engine.engine import LLMEngine
    if mcfg.arch == "vibunex" and device == "cuda" and os.environ.get("DLI_BENCH_VIBUNEX_ON_GPU") != "1":
        # the one run of this stack at these sizes ended in an illegal memory access in a step after the start-up checks;
        # until the kernel is found the GPU run has to be asked for explicitly
        raise RuntimeError("vibunex stacks at these layer sizes faulted a GPU in their last run (kernel not identified): "
                           "set DLI_BENCH_VIBUNEX_ON_GPU=1 to run them anyway, or use --device cpu")
    T = 4096
    pages = batch * ((prompt + new_tokens + 64) // 32 + 1) + 64
    eng = LLMEngine(EngineConfig(model=mcfg, device=device, cache=CacheConfig(num_blocks=pages, enable_prefix_caching=False),
                                 sched=SchedulerConfig(max_num_seqs=batch, max_num_batched_tokens=T, max_model_len=prompt + new_tokens + 8,
                                                       long_prefill_chunk=2048),
                                 use_hip_graphs=graphs, graph_batch_sizes=(batch,), mixed_step_graphs=False, tune_gemms=False))
    if graphs:
        eng.warmup()
    rng = np.random.default_rng(0)

    def prompts(n):
        return [rng.integers(3, mcfg.vocab_size, size=prompt).tolist() for _ in range(n)]

    def sync():
        if device == "cuda":
            torch.cuda.synchronize()

    eng.generate(None, SamplingParams(temperature=0.0, max_tokens=2, ignore_eos=True), prompt_ids=prompts(2))   # warm the eager path
    # ---- prefill: one-token requests
    sync()
    t0 = time.perf_counter()
    eng.generate(None, SamplingParams(temperature=0.0, max_tokens=1, ignore_eos=True), prompt_ids=prompts(batch))
    sync()
    t_prefill = time.perf_counter() - t0
    # ---- decode: from "every request has its first token" to the end
    ps = prompts(batch)
    for i, p in enumerate(ps):
        eng.add_request(f"d{i}", None, SamplingParams(temperature=0.0, max_tokens=new_tokens + 1, ignore_eos=True), p)
    reqs = [eng.requests[f"d{i}"] for i in range(batch)]
    while min(r.num_output - r.pending for r in reqs) < 1:
        eng.step()
    sync()
    done0 = sum(r.num_output for r in reqs)
    t0 = time.perf_counter()
    steps = 0
    while eng.has_unfinished():
        eng.step()
        steps += 1
    sync()
    t_decode = time.perf_counter() - t0
    made = sum(r.num_output for r in reqs) - done0
    return {"model": mcfg.name, "params_per_layer_M": round((mcfg.param_count() - (1 if mcfg.tie_embeddings else 2) * mcfg.vocab_size * mcfg.hidden_size) / LAYERS / 1e6, 1),
            "prompt": prompt, "batch": batch, "prefill_tokens_per_s": round(batch * prompt / t_prefill),
            "prefill_ms": round(t_prefill * 1e3, 2), "decode_tokens_per_s": round(made / t_decode),
            "decode_ms_per_step": round(t_decode / max(steps, 1) * 1e3, 3), "decode_steps": steps,
            "graph_steps": eng.runner.stats["graph_steps"], "dtype": mcfg.dtype}


def main(argv=None, out=None):
    ap = argparse.ArgumentParser(description=__doc__.split("\n\n")[0])
    ap.add_argument("--sizes", default="small,large")
    ap.add_argument("--models", default="llama,rodelix,rodelix-attention,rodelix-lightning,rodelix-latent_attention")
    ap.add_argument("--prompt", type=int, default=2048)
    ap.add_argument("--batch", type=int, default=32)
    ap.add_argument("--new-tokens", type=int, default=64)
    ap.add_argument("--device", default="cuda")
    ap.add_argument("--no-graphs", action="store_true")
    a = ap.parse_args(argv)
    out = out or sys.stdout
    for size in a.sizes.split(","):
        cfgs = model_configs(size)
        for name in a.models.split(","):
            rec = run_one(cfgs[name], a.prompt, a.batch, a.new_tokens, a.device, not a.no_graphs)
            rec["size"] = size
            print(json.dumps(rec), file=out, flush=True)
    return 0


if __name__ == "__main__":
    sys.exit(main())
