"""Plain restatement of the Lebepel decoder for the tests: one short function per mechanism, no batching, no cache, no
chunking -- every position recomputed from the definition, in the floating type of the inputs (tests use float64).
Shares nothing with the product path; a model is ``(cfg, w)`` with the parsed config.json and ``{tensor name: torch tensor}``."""
from __future__ import annotations

import torch


def rms(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def norm(x, w, eps):
    """RMS norm with scale 1 + w."""
    return rms(x, eps) * (1 + w)


def silu(z):
    return z / (1 + torch.exp(-z))


def softplus(z):
    return torch.clamp(z, min=0) + torch.log1p(torch.exp(-z.abs()))


def linear(x, w, b=None):
    y = x @ w.T
    return y if b is None else y + b


def embedding(tokens, embed, pos):
    """Token vector plus the learned vector of its position."""
    t = torch.as_tensor(tokens)
    return embed[t] + pos[torch.arange(len(t))]


def sigmoid_attention(q, k, v, scale, r1, r2, pb, eps):
    """q [T, H, dim], k [T, G, dim], v [T, G, vdim] -> [T, H, vdim].  Per-head unit-RMS queries and keys; a visible key's
    weight is sigmoid(q.k scale - r1 ln(1 + r2 distance) + pb), not normalised over the keys."""
    T, H, _ = q.shape
    rep = H // k.shape[1]
    q, k = rms(q, eps), rms(k, eps)
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    for h in range(H):
        g = h // rep
        for i in range(T):
            j = torch.arange(i + 1)
            s = (k[: i + 1, g] @ q[i, h]) * scale - r1[h] * torch.log1p(r2[h] * (i - j).to(q.dtype))
            out[i, h] = torch.sigmoid(s + pb[h]) @ v[: i + 1, g]
    return out


def attention(h, w, p, mix, eps):
    """The whole mixer on rows h [T, width]; ``p`` = tensor prefix ('l3.mix.')."""
    T = h.shape[0]
    proj = lambda n, heads: linear(h, w[p + n], w[p + n + ".b"]).view(T, heads, -1)
    o = sigmoid_attention(proj("q", mix["heads"]), proj("k", mix["kv_heads"]), proj("v", mix["kv_heads"]), mix["scale"],
                          w[p + "r1"], w[p + "r2"], w[p + "pb"], eps)
    return linear(o.reshape(T, -1), w[p + "o"], w[p + "o.b"])


def short_conv(x, taps, bias):
    """y_t = bias + sum_j taps[:, j] x_{t - (n - 1) + j}, channel by channel; x_s = 0 for s < 0.  x [T, ch], taps [ch, n]."""
    T, n = x.shape[0], taps.shape[1]
    y = torch.zeros_like(x) + bias
    for t in range(T):
        for j in range(n):
            s = t - (n - 1) + j
            if s >= 0:
                y[t] = y[t] + taps[:, j] * x[s]
    return y


def ssm(x, B, C, dt, A_log, D):
    """x [T, heads, P], B / C [T, groups, N], dt [T, heads] (after softplus) -> (y [T, heads, P], final state [heads, N, P])."""
    T, H, P = x.shape
    rep = H // B.shape[1]
    S = torch.zeros(H, B.shape[2], P, dtype=x.dtype)
    y = torch.zeros_like(x)
    for t in range(T):
        for h in range(H):
            S[h] = torch.exp(-torch.exp(A_log[h]) * dt[t, h]) * S[h] + dt[t, h] * torch.outer(B[t, h // rep], x[t, h])
            y[t, h] = S[h].T @ C[t, h // rep] + D[h] * x[t, h]
    return y, S


def gated_group_norm(y, z, w, groups, eps):
    """v = y silu(z); rms over each of ``groups`` slices of v, scaled by w."""
    T = y.shape[0]
    return rms((y * silu(z)).view(T, groups, -1), eps).reshape(T, -1) * w


def mamba2(h, w, p, mix, eps):
    T, H, P, N, G = h.shape[0], mix["heads"], mix["vdim"], mix["state"], mix["groups"]
    inner = H * P
    z, xbc, dt = linear(h, w[p + "in"]).split([inner, inner + 2 * G * N, H], dim=1)
    xbc = silu(short_conv(xbc, w[p + "conv"], w[p + "conv.b"]))
    x, B, C = xbc.split([inner, G * N, G * N], dim=1)
    dt = softplus(dt + w[p + "dt_bias"])
    y, _ = ssm(x.reshape(T, H, P), B.reshape(T, G, N), C.reshape(T, G, N), dt, w[p + "A_log"], w[p + "D"])
    return linear(gated_group_norm(y.reshape(T, inner), z, w[p + "norm"], mix["norm_groups"], eps), w[p + "o"])


def feed_forward(h, w, p):
    return linear(silu(linear(h, w[p + "gate"])) * linear(h, w[p + "up"]), w[p + "down"])


MIXERS = {"attention": attention, "mamba2": mamba2}


def layer_runs(cfg):
    """[(layer, add the embedding output first)] in execution order."""
    n, lp = len(cfg["layers"]), cfg.get("loop")
    if not lp:
        return [(i, False) for i in range(n)]
    runs = [(i, False) for i in range(lp["start"])]
    for p in range(lp["times"]):
        runs += [(i, p > 0 and i == lp["start"]) for i in range(lp["start"], lp["stop"])]
    return runs + [(i, False) for i in range(lp["stop"], n)]


def forward(cfg, w, tokens, dtype=torch.float64, collect=None):
    """Logits [T, vocab] of one sequence; ``collect``: a list that receives the residual stream after every layer run."""
    w = {k: (v.to(dtype) if v.is_floating_point() else v) for k, v in w.items()}
    eps, m = cfg["norm"]["eps"], cfg["residual_mult"]
    x0 = x = embedding(tokens, w["embed"], w["pos"])
    for i, again in layer_runs(cfg):
        lay, p = cfg["layers"][i], f"l{i}."
        if again:
            x = x + x0
        h = norm(x, w[p + "norm1"], eps)
        s = MIXERS[lay["type"]](h, w, p + "mix.", lay["mixer"], eps)
        if lay["mlp"] is not None:
            s = s + feed_forward(h, w, p + "mlp.")
        x = x + m * s
        if collect is not None:
            collect.append(x)
    logits = linear(norm(x, w["final.norm"], eps), w["head"])
    c = cfg["logit_softcap"]
    return c * torch.tanh(logits / c)
