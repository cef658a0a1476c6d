"""Plain float64 implementation of Nefarax stacks, written from the equations: one function per mechanism, whole sequences
at once, token by token, no cache, no batching — and no code shared with the package.  The tests compare the engine with
``forward``.

``faults`` gets single mechanisms wrong on purpose (a test first shows that the oracle tells the difference, then that the
engine agrees with the right one):
``squash`` (norms without the tanh), ``norm_bias`` (norms without their bias), ``mult`` (sublayers added with weight 1),
``stale`` (the feed-forward reads the norm of the stream after the mixer), ``conv`` (convolutions see the current token
only), ``conv_act`` (no silu behind the delta rule's convolutions), ``unit`` (q and k of the delta rule not brought to unit
length), ``beta`` (write strength 1), ``decay`` (states never decay), ``erase`` (the delta rule adds without subtracting what
the key already reads), ``late_read`` (the state is read before the token's write), ``out_norm`` (no per-head norm of a
recurrence's output), ``gate`` (no output gates), ``cap`` (mLSTM gates not capped), ``normaliser`` (mLSTM output not divided), ``rotated_values`` (values are the keys after rotation),
``scaling`` (plain frequencies), ``rotation`` (no rotation), ``sink`` (no sink in the denominator), ``skip`` (no ``D x``
term), ``late_gate`` (the gate comes behind the grouped norm), ``one_group`` (one root mean square over all groups),
``dt_bias`` (no bias of the step size), ``half`` (the side-by-side outputs are summed, not averaged), ``side_norm`` (they are
not normed)."""
from __future__ import annotations

import math

import torch

F64 = torch.float64


# ---------------------------------------------------------------------------------------------- small functions
def tanh_norm(x, alpha, w, b, faults=()):
    z = alpha * x
    if "squash" not in faults:
        z = torch.tanh(z)
    return z * w + (0.0 if "norm_bias" in faults else b)


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def silu(z):
    return z * torch.sigmoid(z)


def softplus(z):
    return torch.clamp(z, min=0.0) + torch.log1p(torch.exp(-z.abs()))


def logsigmoid(z):
    return -softplus(-z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def causal_conv(x, w, b=None, current_only=False):
    """x [T, C]; w [C, taps], last column the current token's; zeros before the start."""
    T, taps = x.shape[0], w.shape[1]
    out = torch.zeros_like(x)
    for j in range(taps):
        back = taps - 1 - j
        if back >= T or (current_only and back):
            continue
        out[back:] += w[:, j] * x[:T - back]
    return out if b is None else out + b


# ---------------------------------------------------------------------------------------------- gated delta rule
def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def delta_scan(q, k, v, g, beta, faults=()):
    """q, k [T, H, D]; v [T, H, Dv]; g, beta [T, H]."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[2], dtype=F64)
    out = torch.zeros_like(v)
    for t in range(T):
        S = g[t][:, None, None] * S
        if "late_read" in faults:
            out[t] = torch.einsum("hde,hd->he", S, q[t])
        seen = 0.0 if "erase" in faults else torch.einsum("hde,hd->he", S, k[t])
        u = beta[t][:, None] * (v[t] - seen)
        S = S + k[t][:, :, None] * u[:, None, :]
        if "late_read" not in faults:
            out[t] = torch.einsum("hde,hd->he", S, q[t])
    return out


def delta_mixer(W, p, m, h, eps, faults=()):
    T = h.shape[0]
    H, G, D, Dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    act = (lambda z: z) if "conv_act" in faults else silu
    q, k, v = (act(causal_conv(h @ W[p + s].T, W[p + s + ".conv"], None, "conv" in faults)) for s in "qkv")
    q, k, v = q.view(T, G, D), k.view(T, G, D), v.view(T, H, Dv)
    if "unit" not in faults:
        q, k = unit(q), unit(k)
    q = q * D ** -0.5
    rep = H // G
    q, k = q.repeat_interleave(rep, dim=1), k.repeat_interleave(rep, dim=1)
    beta = torch.sigmoid(h @ W[p + "b"].T)
    if "beta" in faults:
        beta = torch.ones_like(beta)
    db = 0.0 if "dt_bias" in faults else W[p + "dt_bias"]
    g = torch.exp(-torch.exp(W[p + "A_log"]) * softplus(h @ W[p + "a"].T + db))
    if "decay" in faults:
        g = torch.ones_like(g)
    o = delta_scan(q, k, v, g, beta, faults)
    if "out_norm" not in faults:
        o = rms(o, eps)
    o = o * W[p + "norm"]
    o = o.reshape(T, H * Dv)
    if "gate" not in faults:
        o = o * silu(h @ W[p + "g"].T)
    return o @ W[p + "o"].T


# ---------------------------------------------------------------------------------------------- mLSTM
def mlstm_scan(q, k, v, i, f, faults=()):
    """q, k [T, H, D]; v [T, H, Dv]; log gates i, f [T, H]."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[2], dtype=F64)
    n = torch.zeros(H, D, dtype=F64)
    m = torch.zeros(H, dtype=F64)
    out = torch.zeros_like(v)
    for t in range(T):
        m_new = torch.maximum(f[t] + m, i[t])
        keep, write = torch.exp(f[t] + m - m_new), torch.exp(i[t] - m_new)
        if "decay" in faults:
            keep = torch.ones_like(keep)
        o = torch.einsum("hde,hd->he", S, q[t])
        S = keep[:, None, None] * S + write[:, None, None] * k[t][:, :, None] * v[t][:, None, :]
        n = keep[:, None] * n + write[:, None] * k[t]
        m = m_new
        if "late_read" not in faults:
            o = torch.einsum("hde,hd->he", S, q[t])
        den = torch.maximum((n * q[t]).sum(-1).abs(), torch.exp(-m)) + 1e-6
        out[t] = o if "normaliser" in faults else o / den[:, None]
    return out


def mlstm_mixer(W, p, m, h, eps, faults=()):
    T = h.shape[0]
    H, D, Dv, cap = m["heads"], m["dim"], m["vdim"], m["gate_cap"]
    q = (h @ W[p + "q"].T * D ** -0.5).view(T, H, D)
    k = (h @ W[p + "k"].T).view(T, H, D)
    v = (h @ W[p + "v"].T).view(T, H, Dv)
    i, f = h @ W[p + "i"].T + W[p + "i.b"], h @ W[p + "f"].T + W[p + "f.b"]
    if "cap" not in faults:
        i, f = cap * torch.tanh(i / cap), cap * torch.tanh(f / cap)
    o = mlstm_scan(q, k, v, i, logsigmoid(f), faults)
    if "out_norm" not in faults:
        o = rms(o, eps)
    o = o.reshape(T, H * Dv) * W[p + "norm"]
    if "gate" not in faults:
        o = o * torch.sigmoid(h @ W[p + "g"].T)
    return o @ W[p + "o"].T


# ---------------------------------------------------------------------------------------------- side by side: attention
def frequencies(rot, plain=False):
    dims = rot["dims"]
    out = []
    for i in range(dims // 2):
        f = rot["base"] ** (-2.0 * i / dims)
        sc = rot.get("scaling")
        if sc and not plain:
            wave = 2.0 * math.pi / f
            if wave > sc["original"] / sc["low"]:
                f = f / sc["factor"]
            elif wave >= sc["original"] / sc["high"]:
                s = (sc["original"] / wave - sc["low"]) / (sc["high"] - sc["low"])
                f = (1.0 - s) * f / sc["factor"] + s * f
        out.append(f)
    return out


def rotate(v, rot, plain=False):
    """v [T, heads, D], row = position: entries i and i + dims/2 of every head are a pair."""
    half = rot["dims"] // 2
    a = torch.arange(v.shape[0], dtype=F64)[:, None] * torch.tensor(frequencies(rot, plain), dtype=F64)
    c, s = torch.cos(a)[:, None], torch.sin(a)[:, None]
    x, y = v[..., :half], v[..., half:2 * half]
    return torch.cat([x * c - y * s, y * c + x * s, v[..., 2 * half:]], dim=-1)


def conv_attention(W, p, m, h, faults=()):
    T = h.shape[0]
    H, G, D = m["heads"], m["kv_heads"], m["dim"]
    q, k = (causal_conv(h @ W[p + s].T, W[p + s + ".conv"], None, "conv" in faults) for s in "qk")
    q, k = q.view(T, H, D), k.view(T, G, D)
    v = k
    rot = m.get("rot")
    if rot and "rotation" not in faults:
        q, k = rotate(q, rot, "scaling" in faults), rotate(k, rot, "scaling" in faults)
    if "rotated_values" in faults:
        v = k
    out = torch.zeros(T, H, D, dtype=F64)
    for hd in range(H):
        g = hd // (H // G)
        s = q[:, hd] @ k[:, g].T * m["scale"]
        s = s.masked_fill(torch.ones(T, T, dtype=torch.bool).triu(1), -math.inf)
        top = s.max(-1, keepdim=True).values
        e = torch.exp(s - top)
        den = e.sum(-1, keepdim=True) + (0.0 if "sink" in faults else torch.exp(W[p + "sink"][hd] - top))
        out[:, hd] = (e / den) @ v[:, g]
    return out.reshape(T, H * D) @ W[p + "o"].T


# ---------------------------------------------------------------------------------------------- side by side: Mamba-2
def ssd_scan(x, B, C, dt, A, faults=()):
    """x [T, H, Dv]; B, C [T, H, N]; dt [T, H]; A [H] > 0."""
    T, H, Dv = x.shape
    S = torch.zeros(H, B.shape[2], Dv, dtype=F64)
    out = torch.zeros_like(x)
    for t in range(T):
        keep = torch.ones(H, dtype=F64) if "decay" in faults else torch.exp(-A * dt[t])
        late = torch.einsum("hne,hn->he", S, C[t])
        S = keep[:, None, None] * S + dt[t][:, None, None] * B[t][:, :, None] * x[t][:, None, :]
        out[t] = late if "late_read" in faults else torch.einsum("hne,hn->he", S, C[t])
    return out


def ssd_mixer(W, p, m, h, eps, faults=()):
    T = h.shape[0]
    H, Dv, N, G, NG = m["heads"], m["vdim"], m["state"], m["groups"], m["norm_groups"]
    inner = H * Dv
    z, xbc, dt = torch.split(h @ W[p + "in"].T, [inner, inner + 2 * G * N, H], dim=-1)
    xbc = silu(causal_conv(xbc, W[p + "conv"], W[p + "conv.b"], "conv" in faults))
    x, B, C = torch.split(xbc, [inner, G * N, G * N], dim=-1)
    x = x.view(T, H, Dv)
    B, C = (t.view(T, G, N).repeat_interleave(H // G, dim=1) for t in (B, C))
    dt = softplus(dt + (0.0 if "dt_bias" in faults else W[p + "dt_bias"]))
    y = ssd_scan(x, B, C, dt, torch.exp(W[p + "A_log"]), faults)
    if "skip" not in faults:
        y = y + W[p + "D"][:, None] * x
    y = y.reshape(T, inner)
    gate = 1.0 if "gate" in faults else silu(z)
    if "late_gate" not in faults:
        y = y * gate
    y = rms(y, eps) if "one_group" in faults else rms(y.view(T, NG, inner // NG), eps).reshape(T, inner)
    y = y * W[p + "norm"]
    if "late_gate" in faults:
        y = y * gate
    return y @ W[p + "o"].T


def parallel_mixer(W, p, m, h, eps, faults=()):
    a = conv_attention(W, p + "left.", m["left"], h, faults)
    b = ssd_mixer(W, p + "right.", m["right"], h, eps, faults)
    if "side_norm" not in faults:
        a, b = rms(a, eps), rms(b, eps)
    return (1.0 if "half" in faults else 0.5) * (a * W[p + "left.out"] + b * W[p + "right.out"])


# ---------------------------------------------------------------------------------------------- the stack
def mixer(W, p, L, h, eps, faults=()):
    if L["type"] == "delta":
        return delta_mixer(W, p, L["mixer"], h, eps, faults)
    if L["type"] == "mlstm":
        return mlstm_mixer(W, p, L["mixer"], h, eps, faults)
    return parallel_mixer(W, p, L["mixer"], h, eps, faults)


def forward(cfg, W, tokens, faults=()):
    """(logits [T, vocab], residual stream after every layer [L, T, width]), float64."""
    W = {k: v.to(F64) for k, v in W.items()}
    eps, mult = cfg["norm"]["eps"], cfg["residual_mult"]
    if "mult" in faults:
        mult = 1.0

    def norm(x, name):
        return tanh_norm(x, W[name + ".alpha"].reshape(()), W[name], W[name + ".b"], faults)

    x = W["embed"][torch.tensor(tokens)]
    outs = []
    for li, L in enumerate(cfg["layers"]):
        p = f"l{li}."
        h = norm(x, p + "norm1")
        y = mixer(W, p + "mix.", L, h, eps, faults)
        if L.get("mlp"):
            if "stale" in faults:
                h = norm(x + mult * y, p + "norm1")
            y = y + gelu_tanh(h @ W[p + "mlp.up"].T) @ W[p + "mlp.down"].T
        x = x + mult * y
        outs.append(x)
    return norm(x, "final.norm") @ W["embed"].T, torch.stack(outs)


# ---------------------------------------------------------------------------------------------- random checkpoints
def random_weights(cfg, seed=0):
    """Tensor name → fp32 tensor, as a checkpoint stores them."""
    g = torch.Generator().manual_seed(seed)

    def mat(o, i, gain=1.0):
        return torch.randn(o, i, generator=g) * gain * i ** -0.5

    def vec(n, mean=0.0, std=0.1):
        return mean + std * torch.randn(n, generator=g)

    def taps(c, t):
        return torch.randn(c, t, generator=g) * 0.6

    Wd, V = cfg["width"], cfg["vocab"]
    W = {"embed": torch.randn(V, Wd, generator=g)}

    def norm(name):
        W.update({name: vec(Wd, 1.0), name + ".b": vec(Wd, 0.0, 0.2), name + ".alpha": torch.tensor(0.6 + 0.4 * torch.rand(1, generator=g).item())})

    for li, L in enumerate(cfg["layers"]):
        norm(f"l{li}.norm1")
        p, m, ml = f"l{li}.mix.", L["mixer"], L.get("mlp")
        if L["type"] == "delta":
            H, G, D, Dv, t = m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["conv"]
            W.update({p + "q": mat(G * D, Wd), p + "k": mat(G * D, Wd), p + "v": mat(H * Dv, Wd), p + "q.conv": taps(G * D, t),
                      p + "k.conv": taps(G * D, t), p + "v.conv": taps(H * Dv, t), p + "b": mat(H, Wd), p + "a": mat(H, Wd, 1.5),
                      p + "A_log": vec(H, -1.0, 1.0), p + "dt_bias": vec(H, -1.5, 0.7), p + "norm": vec(Dv, 1.0), p + "g": mat(H * Dv, Wd),
                      p + "o": mat(Wd, H * Dv, 1.5)})
        elif L["type"] == "mlstm":
            H, D, Dv = m["heads"], m["dim"], m["vdim"]
            W.update({p + "q": mat(H * D, Wd, 1.5), p + "k": mat(H * D, Wd, 1.5), p + "v": mat(H * Dv, Wd), p + "g": mat(H * Dv, Wd),
                      p + "i": mat(H, Wd, 2.0), p + "i.b": vec(H, -0.5, 0.5), p + "f": mat(H, Wd, 2.0), p + "f.b": vec(H, 2.0, 1.0),
                      p + "norm": vec(H * Dv, 1.0), p + "o": mat(Wd, H * Dv, 1.5)})
        else:
            a, b = m["left"], m["right"]
            H, G, D, t = a["heads"], a["kv_heads"], a["dim"], a["conv"]
            W.update({p + "left.q": mat(H * D, Wd, 1.5), p + "left.k": mat(G * D, Wd, 1.5), p + "left.q.conv": taps(H * D, t),
                      p + "left.k.conv": taps(G * D, t), p + "left.sink": vec(H, 0.5, 1.0), p + "left.o": mat(Wd, H * D)})
            H, Dv, N, G, t = b["heads"], b["vdim"], b["state"], b["groups"], b["conv"]
            C = H * Dv + 2 * G * N
            W.update({p + "right.in": mat(H * Dv + C + H, Wd), p + "right.conv": taps(C, t), p + "right.conv.b": vec(C, 0.0, 0.2),
                      p + "right.dt_bias": vec(H, -1.5, 0.7), p + "right.A_log": vec(H, -0.5, 1.0), p + "right.D": vec(H, 1.0, 0.3),
                      p + "right.norm": vec(H * Dv, 1.0), p + "right.o": mat(Wd, H * Dv), p + "left.out": vec(Wd, 1.0), p + "right.out": vec(Wd, 1.0)})
        if ml:
            W.update({f"l{li}.mlp.up": mat(ml["ff"], Wd), f"l{li}.mlp.down": mat(Wd, ml["ff"])})
    norm("final.norm")
    return W
