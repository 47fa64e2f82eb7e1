"""Plain, slow implementation of the Rizurax decoder, written from its equations.

One function per mechanism, float64 throughout, whole sequences at once, no cache and no batching.
The tests compare the engine against it; nothing here is imported by the package and nothing of
the package is imported here.

Weights come as a dict name -> tensor with the checkpoint's names: ``embed``, ``bigram``, ``head``, ``final.norm``, and per
layer i ``l<i>.norm1`` (and ``.norm2`` when it has a feed-forward), ``l<i>.mix.*`` and ``l<i>.mlp.*``. The configuration is the
parsed ``config.json`` (a dict).
"""
import math

import torch

F = torch.float64


def rms_norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


def silu(z):
    return z * torch.sigmoid(z)


def gelu_tanh(z):
    return 0.5 * z * (1 + torch.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z ** 3)))


def softplus(z):
    return torch.log1p(torch.exp(-z.abs())) + torch.clamp(z, min=0)


def bigram_rows(tokens, buckets, mul_prev, mul_cur):
    """Table row of each place: the last one for the first token, else a hash of (previous, current)."""
    return [buckets if t == 0 else (int(tokens[t - 1]) * mul_prev + int(tok) * mul_cur) % buckets
            for t, tok in enumerate(tokens)]


def causal_conv(u, w):
    """u [T, C], w [C, taps]: y_t = sum_j w[:, j] u_(t - taps + 1 + j), zeros before the start."""
    T = u.shape[0]
    taps = w.shape[1]
    y = torch.zeros_like(u)
    for t in range(T):
        for j in range(taps):
            s = t - taps + 1 + j
            if s >= 0:
                y[t] += w[:, j] * u[s]
    return y


def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def delta_rule(q, k, v, beta, log_g):
    """q, k [T, H, D], v [T, H, Dv], beta and log_g [T, H] -> [T, H, Dv]: the memory decays, is read at k, corrected
    towards v at k, and read out at q."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[2], dtype=F)
    out = torch.zeros(T, H, v.shape[2], dtype=F)
    for t in range(T):
        S = S * torch.exp(log_g[t])[:, None, None]
        u = beta[t][:, None] * (v[t] - (S * k[t][:, :, None]).sum(1))
        S = S + k[t][:, :, None] * u[:, None, :]
        out[t] = (S * q[t][:, :, None]).sum(1)
    return out


def delta(h, W, p, m, eps):
    T = h.shape[0]
    H, G, D, Dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = [silu(causal_conv(h @ W[p + n].T, W[p + n + ".conv"])) for n in ("q", "k", "v")]
    rep = torch.arange(H) // (H // G)                # q / k head of each head
    q = unit(q.view(T, G, D))[:, rep] * D ** -0.5
    k = unit(k.view(T, G, D))[:, rep]
    beta = torch.sigmoid(h @ W[p + "b"].T)
    log_g = -torch.exp(W[p + "A_log"]) * softplus(h @ W[p + "a"].T + W[p + "dt_bias"])
    o = delta_rule(q, k, v.view(T, H, Dv), beta, log_g)
    o = rms_norm(o, W[p + "norm"], eps) * silu(h @ W[p + "g"].T).view(T, H, Dv)
    return o.reshape(T, H * Dv) @ W[p + "o"].T


def frequencies(rot):
    """Angle per position of each turning pair, and the factor on cosine and sine."""
    dims, base = rot["dims"], rot["base"]
    f = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    s = rot.get("scaling")
    if not s:
        return f, 1.0

    def at(turns):
        return dims * math.log(s["original"] / (2 * math.pi * turns)) / (2 * math.log(base))
    lo, hi = max(math.floor(at(s["fast"])), 0), min(math.ceil(at(s["slow"])), dims - 1)
    out = []
    for i, fi in enumerate(f):
        r = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(fi / s["factor"] * r + fi * (1 - r))
    return out, 0.1 * math.log(s["factor"]) + 1.0


def turn_pairs(x, rot):
    """x [T, ..., D]: neighbours (2i, 2i + 1) of the first ``dims`` coordinates of row t turn by t * f_i."""
    out = x.clone()
    f, mag = frequencies(rot)
    for t in range(x.shape[0]):
        for i, fi in enumerate(f):
            c, s = mag * math.cos(t * fi), mag * math.sin(t * fi)
            u, v = x[t, ..., 2 * i], x[t, ..., 2 * i + 1]
            out[t, ..., 2 * i] = u * c - v * s
            out[t, ..., 2 * i + 1] = v * c + u * s
    return out


def softmax_map(q, k, scale):
    """q, k [T, D] -> causal weights [T, T]."""
    T = q.shape[0]
    s = (q @ k.T) * scale
    return torch.softmax(s.masked_fill(torch.arange(T)[None, :] > torch.arange(T)[:, None], float("-inf")), -1)


def lambda_of(W, p, diff):
    return float(torch.exp((W[p + "lq1"] * W[p + "lk1"]).sum()) - torch.exp((W[p + "lq2"] * W[p + "lk2"]).sum())) + diff


def differential_attention(h, W, p, m, eps, return_weights=False):
    """Two softmax maps per head over the same values, the second taken off the first."""
    T = h.shape[0]
    H, G, D, Dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = turn_pairs((h @ W[p + "q"].T).view(T, H, 2, D), m["rot"])
    k = turn_pairs((h @ W[p + "k"].T).view(T, G, 2, D), m["rot"])
    v = (h @ W[p + "v"].T).view(T, G, Dv)
    lam = lambda_of(W, p, m["diff"])
    o = torch.zeros(T, H, Dv, dtype=F)
    weights = torch.zeros(H, 2, T, T, dtype=F)
    for i in range(H):
        g = i // (H // G)
        for j in range(2):
            weights[i, j] = softmax_map(q[:, i, j], k[:, g, j], m["scale"])
        o[:, i] = weights[i, 0] @ v[:, g] - lam * (weights[i, 1] @ v[:, g])
    o = rms_norm(o, 1.0, eps) * (1 - m["diff"])
    y = o.reshape(T, H * Dv) @ W[p + "o"].T
    return (y, weights) if return_weights else y


def dense_ff(h, W, p):
    return (gelu_tanh(h @ W[p + "gate"].T) * (h @ W[p + "up"].T)) @ W[p + "down"].T


def layer_runs(cfg):
    n = len(cfg["layers"])
    loop = cfg.get("loop")
    if not loop:
        return list(range(n))
    a, b = loop["start"], loop["stop"]
    return list(range(a)) + list(range(a, b)) * loop["times"] + list(range(max(a, b), n))


def forward(cfg, W, tokens, return_layers=False):
    """Logits [T, vocab] (float64) of a whole sequence; with ``return_layers`` also the stream after every layer run."""
    W = {k: v.to(F) for k, v in W.items()}
    eps = cfg["norm"]["eps"]
    x = W["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    big = (cfg.get("embedding") or {}).get("bigram")
    if big:
        x = x + W["bigram"][bigram_rows(tokens, big["buckets"], big["mul_prev"], big["mul_cur"])]
    taps = []
    for i in layer_runs(cfg):
        L, p = cfg["layers"][i], f"l{i}."
        mixer = {"delta": delta, "attention": differential_attention}[L["type"]]
        y = mixer(rms_norm(x, 1 + W[p + "norm1"], eps), W, p + "mix.", L["mixer"], eps)
        if L.get("mlp") is not None:
            y = y + dense_ff(rms_norm(x, 1 + W[p + "norm2"], eps), W, p + "mlp.")
        x = x + y
        taps.append(x)
    logits = rms_norm(x, 1 + W["final.norm"], eps) @ W["head"].T
    return (logits, taps) if return_layers else logits


def random_weights(cfg, seed=0):
    """bf16 tensors under the checkpoint's names: matrices N(0, 1 / fan_in) (queries and keys of the attention larger, so
    that the softmax is not flat), offset norm weights far from zero, decays from a token's to hundreds of tokens' memory."""
    gen = torch.Generator().manual_seed(seed)
    d, V = cfg["width"], cfg["vocab"]
    W = {}

    def mat(n, k, s=1.0):
        return (torch.randn(n, k, generator=gen) * s * k ** -0.5).to(torch.bfloat16)

    def vec(n, mean=0.0, s=0.1):
        return (mean + s * torch.randn(n, generator=gen)).to(torch.bfloat16)
    W["embed"] = mat(V, d, d ** 0.5)
    big = (cfg.get("embedding") or {}).get("bigram")
    if big:
        W["bigram"] = mat(big["buckets"] + 1, d, d ** 0.5)
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        x = p + "mix."
        W[p + "norm1"] = vec(d, s=0.3)
        H, G, D, Dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        if L["type"] == "delta":
            for n, c in (("q", G * D), ("k", G * D), ("v", H * Dv)):
                W[x + n] = mat(c, d, 1.5)
                W[x + n + ".conv"] = (torch.randn(c, m["conv"], generator=gen) * 0.6).to(torch.bfloat16)
            W[x + "b"], W[x + "a"], W[x + "g"], W[x + "o"] = mat(H, d, 2.0), mat(H, d), mat(H * Dv, d, 1.5), mat(d, H * Dv)
            W[x + "A_log"] = torch.linspace(-1.0, 1.5, H).to(torch.bfloat16)
            W[x + "dt_bias"] = torch.linspace(-5.0, 0.5, H)[torch.randperm(H, generator=gen)].to(torch.bfloat16)
            W[x + "norm"] = vec(Dv, 1.0, 0.3)
        else:
            W[x + "q"], W[x + "k"] = mat(H * 2 * D, d, 2.0), mat(G * 2 * D, d, 2.0)
            W[x + "v"], W[x + "o"] = mat(G * Dv, d), mat(d, H * Dv)
            for n in ("lq1", "lk1", "lq2", "lk2"):
                W[x + n] = vec(D, s=0.3)
        if L.get("mlp") is not None:
            n = L["mlp"]["ff"]
            W[p + "norm2"] = vec(d, s=0.3)
            f = p + "mlp."
            W[f + "gate"], W[f + "up"], W[f + "down"] = mat(n, d, 1.5), mat(n, d, 1.5), mat(d, n)
    W["final.norm"], W["head"] = vec(d, s=0.3), mat(V, d)
    return W
