"""Plain restatement of the Serotar decoder for the tests: one short function per mechanism, no batching, no cache, no portions -- every
position recomputed from the definition, in the floating type of the inputs (tests use float64).  Shares nothing with the product path; a model
is ``(cfg, w)`` with the parsed config.json and ``{tensor name: torch tensor}``."""
from __future__ import annotations

import math

import torch


def rms(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def linear(x, w):
    return x @ w.T


def silu(z):
    return z / (1 + torch.exp(-z))


def softplus(z):
    return torch.clamp(z, min=0) + torch.log1p(torch.exp(-z.abs()))


def gelu_tanh(z):
    return 0.5 * z * (1 + torch.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z ** 3)))


def xielu(z, p, q):
    """Quadratic above zero, exponential below, slope 1/2 at zero."""
    up = softplus(p) * z * z + 0.5 * z
    down = (0.5 + softplus(q)) * (torch.exp(torch.clamp(z, max=0)) - 1 - z) + 0.5 * z
    return torch.where(z > 0, up, down)


def bigram_rows(tokens, bg):
    """Row of the bigram table at every position; the extra last row opens a sequence."""
    return [bg["buckets"]] + [(a * bg["mul_prev"] + b * bg["mul_cur"]) % bg["buckets"] for a, b in zip(tokens, tokens[1:])]


def embedding(cfg, w, tokens):
    e = cfg["embedding"]
    x = w["embed"][torch.as_tensor(tokens)] * e["scale"]
    if e.get("bigram"):
        x = x + w["bigram"][torch.as_tensor(bigram_rows(list(tokens), e["bigram"]))]
    return x


def softmax_attention(q, k, v, scale):
    """Causal.  q, k [T, H, dim], v [T, H, vdim] -> [T, H, vdim]."""
    T = q.shape[0]
    out = torch.zeros(T, q.shape[1], v.shape[2], dtype=q.dtype)
    hide = torch.triu(torch.ones(T, T, dtype=torch.bool), diagonal=1)
    for h in range(q.shape[1]):
        s = (q[:, h] @ k[:, h].T) * scale
        s = s.masked_fill(hide, -math.inf)
        a = torch.exp(s - s.max(-1, keepdim=True).values)
        out[:, h] = (a / a.sum(-1, keepdim=True)) @ v[:, h]
    return out


def latent_attention(h, w, p, mix, eps):
    """The whole mixer on rows h [T, width]; ``p`` = tensor prefix ('l3.mix.')."""
    T, H = h.shape[0], mix["heads"]
    cq = rms(linear(h, w[p + "dq"]), eps) * w[p + "dq.norm"]
    c = rms(linear(h, w[p + "dkv"]), eps) * w[p + "dkv.norm"]
    o = softmax_attention(linear(cq, w[p + "uq"]).view(T, H, -1), linear(c, w[p + "uk"]).view(T, H, -1), linear(c, w[p + "uv"]).view(T, H, -1), mix["scale"])
    return linear(o.reshape(T, -1), w[p + "o"])


def dense_ff(h, w, p):
    a = w[p + "act"]
    return linear(xielu(linear(h, w[p + "up"]), a[0], a[1]), w[p + "down"])


def expert(h, w, p):
    return linear(silu(linear(h, w[p + "gate"])) * linear(h, w[p + "up"]), w[p + "down"])


def choose(s, correction, router):
    """Indices of the experts one token uses, from its scores s [experts + identity]."""
    choice = (s + correction).tolist()
    n = len(choice)
    allowed = range(n)
    if router.get("groups"):
        size = n // router["groups"]["count"]
        best = sorted(range(router["groups"]["count"]), key=lambda g: -max(choice[g * size:(g + 1) * size]))[:router["groups"]["keep"]]
        allowed = [i for i in range(n) if i // size in best]
    return sorted(allowed, key=lambda i: -choice[i])[:router["top"]]


def mixture(h, w, p, mlp):
    r = mlp["router"]
    s = torch.softmax(linear(h, w[p + "router"]), -1)
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for i in choose(s[t], w[p + "correction"], r):
            out[t] += s[t, i] * (h[t] if i >= r["experts"] else expert(h[t], w, p + f"e{i}."))
    if mlp.get("shared"):
        out = out + expert(h, w, p + "shared.")
    return out


def feed_forward(h, w, p, mlp):
    return dense_ff(h, w, p) if mlp["kind"] == "dense" else mixture(h, w, p, mlp)


def token_side(x, tokens, i, w, dim, eps):
    e = w["side.embed"][torch.as_tensor(tokens)][:, i * dim:(i + 1) * dim]
    y = linear(gelu_tanh(linear(x, w[f"l{i}.side.gate"])) * e, w[f"l{i}.side.proj"])
    return x + rms(y, eps) * w[f"l{i}.side.norm"]


def forward(cfg, w, tokens, dtype=torch.float64, collect=None):
    """Logits [T, vocab] of one sequence; ``collect``: a list that receives the residual stream after every layer."""
    w = {k: (v.to(dtype) if v.is_floating_point() else v) for k, v in w.items()}
    eps = cfg["norm"]["eps"]
    x = embedding(cfg, w, tokens)
    X = [x]
    for i, lay in enumerate(cfg["layers"]):
        p = f"l{i}."
        x = x + rms(latent_attention(x, w, p + "mix.", lay["mixer"], eps), eps) * w[p + "norm1"] * w[p + "ls1"]
        if lay["mlp"] is not None:
            x = x + rms(feed_forward(x, w, p + "mlp.", lay["mlp"]), eps) * w[p + "norm2"] * w[p + "ls2"]
        if cfg.get("token_side"):
            x = token_side(x, tokens, i, w, cfg["token_side"]["dim"], eps)
        X.append(x)
        x = sum(w[p + "dwa"][j] * X[j] for j in range(i + 2))
        if collect is not None:
            collect.append(x)
    return linear(rms(x, eps) * w["final.norm"], w["head"])
