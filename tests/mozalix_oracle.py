"""Plain float64 implementation of Mozalix stacks, written from the equations: one function per mechanism, whole sequences
at once, token by token, no cache, no batching — and no code shared with the package.  The tests compare the engine with
``forward``.

``faults`` gets single mechanisms wrong on purpose (a test first shows that the oracle tells the difference, then that the
engine agrees with the right one):
``embed_scale`` (rows of the table unscaled), ``norm_offset`` (stream norms times ``w`` instead of ``1 + w``), ``pre_norm`` (the
feed-forward reads the normed mixer output instead of the stream), ``shared`` (a layer on another's weights runs without its
feed-forward), ``qk_norm`` (queries and keys not normed), ``qk_weight`` (their norm without its weight), ``late_norm`` (normed
behind the rotation), ``rotation`` (no rotation), ``chunk`` (no chunk edges), ``chunk_size`` (one too wide), ``sink`` (no sink),
``window`` (one too wide), ``narrow`` (one too narrow), ``keep`` (no kept first tokens), ``keep_more`` (one more kept), ``softcap``
(none), ``one_map`` (the second map not subtracted), ``lambda`` (without the exponentials' difference), ``map_norm`` (the difference of the
maps not normed), ``map_scale`` (nor scaled), ``map_heads`` (the second map reads the first one's keys), ``scales`` (the halves
summed with weight 1), ``conv`` (convolutions see the current token only), ``conv_act`` (no silu behind them), ``unit`` (q and k of
the delta rule not brought to unit length), ``q_scale`` (its queries not scaled), ``beta`` (write strength 1), ``decay`` (states
never decay), ``head_decay`` (one decay per head: the mean over its key channels), ``erase`` (the delta rule adds without
subtracting what the key already reads), ``late_read`` (the state is read before the token's write), ``dt_bias`` (no bias of the
decay), ``out_norm`` (no per-head norm of the recurrence's output), ``gate`` (no output gate), ``limit`` (feed-forward not clamped),
``up_offset`` (``u`` instead of ``u + 1``), ``gate_slope`` (``sigmoid(g)``), ``ff_bias`` (no biases)."""
from __future__ import annotations

import math

import torch

F64 = torch.float64


# ---------------------------------------------------------------------------------------------- small functions
def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def stream_norm(x, w, eps, faults=()):
    return rms(x, eps) * (w if "norm_offset" in faults else 1.0 + w)


def silu(z):
    return z * torch.sigmoid(z)


def softplus(z):
    return torch.clamp(z, min=0.0) + torch.log1p(torch.exp(-z.abs()))


def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def causal_conv(x, w, current_only=False):
    """x [T, C]; w [C, taps], last column the current token's; zeros before the start."""
    T, taps = x.shape[0], w.shape[1]
    out = torch.zeros_like(x)
    for j in range(taps):
        back = taps - 1 - j
        if back >= T or (current_only and back):
            continue
        out[back:] += w[:, j] * x[:T - back]
    return out


def rotate(v, rot):
    """v [T, ..., D], row = position: entries i and i + dims/2 of the last axis are a pair."""
    dims, half = rot["dims"], rot["dims"] // 2
    f = torch.tensor([rot["base"] ** (-2.0 * i / dims) for i in range(half)], dtype=F64)
    a = torch.arange(v.shape[0], dtype=F64).reshape([-1] + [1] * (v.dim() - 1)) * f
    c, s = torch.cos(a), torch.sin(a)
    x, y = v[..., :half], v[..., half:dims]
    return torch.cat([x * c - y * s, y * c + x * s, v[..., dims:]], dim=-1)


# ---------------------------------------------------------------------------------------------- who sees whom
def visible(T, kind, mask, faults=()):
    """bool [T, T]: row i sees column j."""
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    causal = j <= i
    if kind == "chunk":
        size = mask["size"] + ("chunk_size" in faults)
        return causal if "chunk" in faults else causal & (torch.div(i, size, rounding_mode="floor") == torch.div(j, size, rounding_mode="floor"))
    size = mask["size"] + ("window" in faults) - ("narrow" in faults)
    near = i - j < size
    if kind == "keep" and "keep" not in faults:
        near = near | (j < mask["keep_first"] + ("keep_more" in faults))
    return causal & near


def softmax_attention(q, k, v, scale, see, cap=None, sink=None):
    """q [T, H, D]; k [T, G, D]; v [T, G, Dv]; see bool [T, T]; sink [H]."""
    T, H = q.shape[:2]
    out = torch.zeros(T, H, v.shape[2], dtype=F64)
    for h in range(H):
        g = h // (H // k.shape[1])
        s = q[:, h] @ k[:, g].T * scale
        if cap is not None:
            s = cap * torch.tanh(s / cap)
        s = s.masked_fill(~see, -math.inf)
        top = s.max(-1, keepdim=True).values
        e = torch.exp(s - top)
        den = e.sum(-1, keepdim=True)
        if sink is not None:
            den = den + torch.exp(sink[h] - top)
        out[:, h] = (e / den) @ v[:, g]
    return out


def normed_qk(W, p, q, k, rot, eps, faults=()):
    """Per-head norm with a weight shared by the heads (none stored: without), then rotation."""
    def one(x, name):
        w = W.get(p + name + ".norm")
        if w is None or "qk_weight" in faults:
            w = 1.0
        x = x if "qk_norm" in faults else rms(x, eps)
        if "late_norm" in faults and rot:
            return rms(rotate(x * w, rot) * w, eps)
        x = x * w
        return rotate(x, rot) if rot and "rotation" not in faults else x
    return one(q, "q"), one(k, "k")


# ---------------------------------------------------------------------------------------------- mixers
def chunk_attention(W, p, m, h, eps, faults=()):
    T = h.shape[0]
    H, G, D, Dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k = normed_qk(W, p, (h @ W[p + "q"].T).view(T, H, D), (h @ W[p + "k"].T).view(T, G, D), m.get("rot"), eps, faults)
    o = softmax_attention(q, k, (h @ W[p + "v"].T).view(T, G, Dv), m["scale"], visible(T, "chunk", m["mask"], faults),
                          sink=None if "sink" in faults else W[p + "sink"])
    return o.reshape(T, H * Dv) @ W[p + "o"].T


def differential_attention(W, p, m, h, eps, faults=()):
    T = h.shape[0]
    H, G, D, Dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k = normed_qk(W, p, (h @ W[p + "q"].T).view(T, H, 2, D), (h @ W[p + "k"].T).view(T, G, 2, D), m.get("rot"), eps, faults)
    v = (h @ W[p + "v"].T).view(T, G, Dv)
    see = visible(T, "window", m["mask"], faults)
    a1 = softmax_attention(q[:, :, 0], k[:, :, 0], v, m["scale"], see)
    a2 = softmax_attention(q[:, :, 1], k[:, :, 0 if "map_heads" in faults else 1], v, m["scale"], see)
    lam = torch.exp((W[p + "lq1"] * W[p + "lk1"]).sum()) - torch.exp((W[p + "lq2"] * W[p + "lk2"]).sum()) + m["diff"]
    if "lambda" in faults:
        lam = m["diff"]
    o = a1 if "one_map" in faults else a1 - lam * a2
    if "map_norm" not in faults:
        o = rms(o, eps)
    if "map_scale" not in faults:
        o = o * (1.0 - m["diff"])
    return o.reshape(T, H * Dv) @ W[p + "o"].T


def capped_attention(W, p, m, h, eps, faults=()):
    T = h.shape[0]
    H, G, D, Dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k = normed_qk({}, p, (h @ W[p + "q"].T).view(T, H, D), (h @ W[p + "k"].T).view(T, G, D), None, eps, faults)
    o = softmax_attention(q, k, (h @ W[p + "v"].T).view(T, G, Dv), m["scale"], visible(T, "keep", m["mask"], faults),
                          cap=None if "softcap" in faults else m["softcap"])
    return o.reshape(T, H * Dv) @ W[p + "o"].T


def channel_delta_scan(q, k, v, g, beta, faults=()):
    """q, k, g [T, H, D]; v [T, H, Dv]; beta [T, H]: the decay acts on the state's rows."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[2], dtype=F64)
    out = torch.zeros_like(v)
    for t in range(T):
        S = g[t][:, :, None] * S
        if "late_read" in faults:
            out[t] = torch.einsum("hde,hd->he", S, q[t])
        seen = 0.0 if "erase" in faults else torch.einsum("hde,hd->he", S, k[t])
        u = beta[t][:, None] * (v[t] - seen)
        S = S + k[t][:, :, None] * u[:, None, :]
        if "late_read" not in faults:
            out[t] = torch.einsum("hde,hd->he", S, q[t])
    return out


def channel_delta(W, p, m, h, eps, faults=()):
    T = h.shape[0]
    H, G, D, Dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    act = (lambda z: z) if "conv_act" in faults else silu
    q, k, v = (act(causal_conv(h @ W[p + s].T, W[p + s + ".conv"], "conv" in faults)) for s in "qkv")
    q, k, v = q.view(T, G, D), k.view(T, G, D), v.view(T, H, Dv)
    if "unit" not in faults:
        q, k = unit(q), unit(k)
    if "q_scale" not in faults:
        q = q * D ** -0.5
    q, k = q.repeat_interleave(H // G, dim=1), k.repeat_interleave(H // G, dim=1)
    beta = torch.sigmoid(h @ W[p + "b"].T)
    if "beta" in faults:
        beta = torch.ones_like(beta)
    z = h @ W[p + "a1"].T @ W[p + "a2"].T + (0.0 if "dt_bias" in faults else W[p + "dt_bias"].reshape(-1))
    log_g = -torch.exp(W[p + "A_log"])[:, None] * softplus(z).view(T, H, D)
    if "head_decay" in faults:
        log_g = log_g.mean(-1, keepdim=True).expand(T, H, D)
    g = torch.ones(T, H, D, dtype=F64) if "decay" in faults else torch.exp(log_g)
    o = channel_delta_scan(q, k, v, g, beta, faults)
    if "out_norm" not in faults:
        o = rms(o, eps)
    o = (o * W[p + "norm"]).reshape(T, H * Dv)
    if "gate" not in faults:
        o = o * torch.sigmoid(h @ W[p + "g1"].T @ W[p + "g2"].T)
    return o @ W[p + "o"].T


def mixer(W, p, L, h, eps, faults=()):
    m = L["mixer"]
    if L["type"] == "attention":
        return chunk_attention(W, p, m, h, eps, faults)
    if L["type"] == "attention_2":
        return differential_attention(W, p, m, h, eps, faults)
    a, b = (1.0, 1.0) if "scales" in faults else (m["left_scale"], m["right_scale"])
    return a * capped_attention(W, p + "left.", m["left"], h, eps, faults) + b * channel_delta(W, p + "right.", m["right"], h, eps, faults)


def feed_forward(W, p, ml, h, faults=()):
    b = {s: 0.0 if "ff_bias" in faults else W[p + s + ".b"] for s in ("gate", "up", "down")}
    g, u = h @ W[p + "gate"].T + b["gate"], h @ W[p + "up"].T + b["up"]
    if "limit" not in faults:
        g, u = torch.clamp(g, max=ml["limit"]), torch.clamp(u, -ml["limit"], ml["limit"])
    y = g * torch.sigmoid((1.0 if "gate_slope" in faults else 1.702) * g) * (u + (0.0 if "up_offset" in faults else 1.0))
    return y @ W[p + "down"].T + b["down"]


# ---------------------------------------------------------------------------------------------- the stack
def forward(cfg, W, tokens, faults=()):
    """(logits [T, vocab], residual stream after every layer [L, T, width]), float64."""
    W = {k: v.to(F64) for k, v in W.items()}
    eps = cfg["norm"]["eps"]
    x = W["embed"][torch.tensor(tokens)] * (1.0 if "embed_scale" in faults else cfg["embedding"]["scale"])
    outs = []
    for li, L in enumerate(cfg["layers"]):
        src = L.get("weights_of")
        p = f"l{li if src is None else src}."
        y = stream_norm(mixer(W, p + "mix.", L, x, eps, faults), W[p + "norm1"], eps, faults)
        x = x + y
        if L.get("mlp") and not ("shared" in faults and src is not None):
            x = x + stream_norm(feed_forward(W, p + "mlp.", L["mlp"], y if "pre_norm" in faults else x, faults), W[p + "norm2"], eps, faults)
        outs.append(x)
    return stream_norm(x, W["final.norm"], eps, faults) @ W["head"].T, torch.stack(outs)


# ---------------------------------------------------------------------------------------------- random checkpoints
def random_weights(cfg, seed=0, ranks=(6, 10)):
    """Tensor name → fp32 tensor, as a checkpoint stores them.  ``ranks``: of the decay's and the output gate's low-rank maps."""
    gen = torch.Generator().manual_seed(seed)

    def mat(o, i, gain=1.0):
        return torch.randn(o, i, generator=gen) * gain * i ** -0.5

    def vec(n, mean=0.0, std=0.1):
        return mean + std * torch.randn(n, generator=gen)

    Wd, V = cfg["width"], cfg["vocab"]
    W = {"embed": torch.randn(V, Wd, generator=gen), "head": mat(V, Wd)}
    for li, L in enumerate(cfg["layers"]):
        if L.get("weights_of") is not None:
            continue
        p, m, ml = f"l{li}.mix.", L["mixer"], L.get("mlp")
        W[f"l{li}.norm1"] = vec(Wd, 0.0, 0.2)
        if L["type"] == "attention":
            H, G, D, Dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
            W.update({p + "q": mat(H * D, Wd), p + "k": mat(G * D, Wd), p + "v": mat(G * Dv, Wd), p + "q.norm": vec(D, 1.3, 0.3),
                      p + "k.norm": vec(D, 1.3, 0.3), p + "sink": vec(H, 0.5, 1.0), p + "o": mat(Wd, H * Dv)})
        elif L["type"] == "attention_2":
            H, G, D, Dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
            W.update({p + "q": mat(H * 2 * D, Wd), p + "k": mat(G * 2 * D, Wd), p + "v": mat(G * Dv, Wd), p + "q.norm": vec(D, 1.3, 0.3),
                      p + "k.norm": vec(D, 1.3, 0.3), p + "o": mat(Wd, H * Dv)})
            W.update({p + s: vec(D, 0.0, 0.55 * D ** -0.25) for s in ("lq1", "lk1", "lq2", "lk2")})
        else:
            a, b = m["left"], m["right"]
            H, G, D, Dv = a["heads"], a["kv_heads"], a["dim"], a["vdim"]
            W.update({p + "left.q": mat(H * D, Wd), p + "left.k": mat(G * D, Wd), p + "left.v": mat(G * Dv, Wd), p + "left.o": mat(Wd, H * Dv)})
            H, G, D, Dv, t = b["heads"], b["kv_heads"], b["dim"], b["vdim"], b["conv"]
            p += "right."
            W.update({p + "q": mat(G * D, Wd), p + "k": mat(G * D, Wd), p + "v": mat(H * Dv, Wd)})
            W.update({p + s + ".conv": torch.randn(n, t, generator=gen) * 0.6 for s, n in (("q", G * D), ("k", G * D), ("v", H * Dv))})
            W.update({p + "b": mat(H, Wd), p + "A_log": vec(H, -1.0, 1.0), p + "dt_bias": vec(H * D, -1.5, 0.7), p + "a1": mat(ranks[0], Wd),
                      p + "a2": mat(H * D, ranks[0], 1.5), p + "g1": mat(ranks[1], Wd), p + "g2": mat(H * Dv, ranks[1]), p + "norm": vec(Dv, 1.0),
                      p + "o": mat(Wd, H * Dv, 1.5)})
        if ml:
            F, p = ml["ff"], f"l{li}.mlp."
            W.update({f"l{li}.norm2": vec(Wd, 0.0, 0.2), p + "gate": mat(F, Wd), p + "up": mat(F, Wd), p + "down": mat(Wd, F),
                      p + "gate.b": vec(F, 0.0, 0.5), p + "up.b": vec(F, 0.0, 0.5), p + "down.b": vec(Wd, 0.0, 0.3)})
    W["final.norm"] = vec(Wd, 0.0, 0.2)
    return W
