"""Plain, slow implementation of the Kulivik decoder, written from its equations.

One function per mechanism, float64 throughout, whole sequences at once, no cache and no batching.
The tests compare the engine against it; nothing here is imported by the package and nothing of
the package is imported here.

Weights come as a dict name -> tensor with the checkpoint's names: ``embed``, ``final.norm``, and per
layer i ``l<i>.norm1``, ``.norm1b``, ``.shift``, ``.rg1``, ``.rg1.b`` (and ``.norm2``, ``.norm2b``, ``.rg2``,
``.rg2.b`` when it has a feed-forward), ``l<i>.mix.*`` and ``l<i>.mlp.*``. The configuration is the
parsed ``config.json`` (a dict).
"""
import math

import torch

F = torch.float64


def rms_norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


def silu(z):
    return z * torch.sigmoid(z)


def token_shift(h, mu):
    """Row t moves towards row t - 1 (zeros before the first row) by ``mu``, element by element."""
    prev = torch.cat([torch.zeros_like(h[:1]), h[:-1]], 0)
    return h + (prev - h) * mu


def causal_conv(u, w):
    """u [T, C], w [C, taps]: y_t = sum_j w[:, j] u_(t - taps + 1 + j), zeros before the start."""
    T, C = u.shape
    taps = w.shape[1]
    y = torch.zeros_like(u)
    for t in range(T):
        for j in range(taps):
            s = t - taps + 1 + j
            if s >= 0:
                y[t] += w[:, j] * u[s]
    return y


def turn_pairs(x, dims, base):
    """x [T, heads, D]: neighbours (2i, 2i + 1) of the first ``dims`` coordinates of row t turn by t * base^(-2i / dims)."""
    out = x.clone()
    for t in range(x.shape[0]):
        for i in range(dims // 2):
            a = t * base ** (-2.0 * i / dims)
            u, v = x[t, :, 2 * i], x[t, :, 2 * i + 1]
            out[t, :, 2 * i] = u * math.cos(a) - v * math.sin(a)
            out[t, :, 2 * i + 1] = v * math.cos(a) + u * math.sin(a)
    return out


def temperature(T, coef, every):
    """The factor on the query of each position."""
    return torch.tensor([1.0 + coef * math.log((p + 1) // every + 1) for p in range(T)], dtype=F)


def head_slopes(H):
    return [2.0 ** (-8.0 * (h + 1) / H) for h in range(H)]


def visible(T, size=0, keep=0):
    """mask[i, j]: row i sees key j. ``size`` > 0: only the last ``size`` positions, or the first ``keep``."""
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    ok = j <= i
    return ok & ((i - j < size) | (j < keep)) if size else ok


def attend(q, k, v, scale, mask, cap=0.0, slopes=None, sink=None):
    """q [T, H, D], k [T, G, D], v [T, G, Dv] -> ([T, H, Dv], weights [H, T, T])."""
    T, H, _ = q.shape
    rep = H // k.shape[1]
    out = torch.zeros(T, H, v.shape[2], dtype=F)
    weights = torch.zeros(H, T, T, dtype=F)
    dist = (torch.arange(T)[:, None] - torch.arange(T)[None, :]).to(F)
    for h in range(H):
        s = (q[:, h] @ k[:, h // rep].T) * scale
        if slopes is not None:
            s = s - slopes[h] * dist
        if cap:
            s = cap * torch.tanh(s / cap)
        s = s.masked_fill(~mask, float("-inf"))
        m = s.max(-1, keepdim=True).values
        if sink is not None:
            m = torch.clamp(m, min=float(sink[h]))
        e = torch.exp(s - m)
        den = e.sum(-1, keepdim=True)
        if sink is not None:
            den = den + torch.exp(sink[h] - m)
        weights[h] = e / den
        out[:, h] = weights[h] @ v[:, h // rep]
    return out, weights


def mixed_values(v, W, p, m, shared):
    """``shared``: a dict that carries the first mixing layer's values through the forward pass."""
    if not m.get("v_mix"):
        return v
    if "v" not in shared:
        shared["v"] = v
        return v
    lam = W[p + "vmix"]
    return (1 - lam) * v + lam * shared["v"]


def conv_attention(h, W, p, m, eps, shared, return_weights=False):
    """Convolved projections, norms over the whole projections, no positions, a learned sink, a gate per head."""
    T = h.shape[0]
    H, G, D, Dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = [causal_conv(h @ W[p + n].T, W[p + n + ".conv"]) for n in ("q", "k", "v")]
    q = rms_norm(q, W[p + "q.norm"], eps).view(T, H, D)
    k = rms_norm(k, W[p + "k.norm"], eps).view(T, G, D)
    v = mixed_values(v, W, p, m, shared).view(T, G, Dv)
    o, w = attend(q, k, v, m["scale"], visible(T), sink=W[p + "sink"])
    o = o * torch.sigmoid(h @ W[p + "g"].T)[:, :, None]
    y = o.reshape(T, H * Dv) @ W[p + "o"].T
    return (y, w) if return_weights else y


def window_attention(h, W, p, m, eps, shared, return_weights=False):
    """Biased projections, norms per head, neighbouring pairs turn, capped scores, a window with kept first tokens."""
    T = h.shape[0]
    H, G, D, Dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = [h @ W[p + n].T + W[p + n + ".b"] for n in ("q", "k", "v")]
    q = rms_norm(q.view(T, H, D), W[p + "q.norm"], eps)
    k = rms_norm(k.view(T, G, D), W[p + "k.norm"], eps)
    rot = m["rot"]
    q, k = turn_pairs(q, rot["dims"], rot["base"]), turn_pairs(k, rot["dims"], rot["base"])
    v = mixed_values(v, W, p, m, shared).view(T, G, Dv)
    o, w = attend(q, k, v, m["scale"], visible(T, m["mask"]["size"], m["mask"].get("keep_first", 0)), cap=m["softcap"])
    y = o.reshape(T, H * Dv) @ W[p + "o"].T + W[p + "o.b"]
    return (y, w) if return_weights else y


def distance_attention(h, W, p, m, return_weights=False):
    """No rotation: a query temperature that grows with the position and a bias per unit of distance."""
    T = h.shape[0]
    H, G, D, Dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (h @ W[p + "q"].T).view(T, H, D), (h @ W[p + "k"].T).view(T, G, D), (h @ W[p + "v"].T).view(T, G, Dv)
    q = q * temperature(T, m["q_temp"]["coef"], m["q_temp"]["every"])[:, None, None]
    o, w = attend(q, k, v, m["scale"], visible(T), slopes=head_slopes(H))
    y = o.reshape(T, H * Dv) @ W[p + "o"].T
    return (y, w) if return_weights else y


def lightning(h, W, p, m, eps):
    """Linear attention with one constant decay per head."""
    T = h.shape[0]
    H, D, Dv = m["heads"], m["dim"], m["vdim"]
    q, k = silu(h @ W[p + "q"].T).view(T, H, D), silu(h @ W[p + "k"].T).view(T, H, D)
    v = silu(h @ W[p + "v"].T).view(T, H, Dv)
    a = torch.tensor(m["decay"], dtype=F)[:, None, None]
    S = torch.zeros(H, D, Dv, dtype=F)
    o = torch.zeros(T, H, Dv, dtype=F)
    for t in range(T):
        S = a * S + k[t][:, :, None] * v[t][:, None, :]
        o[t] = (S * q[t][:, :, None]).sum(1)
    o = rms_norm(o.reshape(T, H * Dv), W[p + "norm"], eps) * torch.sigmoid(h @ W[p + "g"].T)
    return o @ W[p + "o"].T


def parallel(h, W, p, m, eps):
    return m["left_scale"] * distance_attention(h, W, p + "left.", m["left"]) + \
        m["right_scale"] * lightning(h, W, p + "right.", m["right"], eps)


def clamped_ff(h, W, p, limit):
    g = torch.clamp(h @ W[p + "gate"].T, max=limit)
    u = torch.clamp(h @ W[p + "up"].T, -limit, limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1)) @ W[p + "down"].T


def routed_ff(h, W, p, mlp):
    z = h @ W[p + "router"].T + W[p + "router.b"]
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        ids = torch.argsort(z[t], descending=True, stable=True)[:mlp["router"]["top"]]
        w = torch.softmax(z[t, ids], 0)
        for e, we in zip(ids.tolist(), w):
            x = f"{p}e{e}."
            out[t] += we * ((silu(W[x + "gate"] @ h[t]) * (W[x + "up"] @ h[t])) @ W[x + "down"].T)
    return out


def forward(cfg, W, tokens, return_layers=False):
    """Logits [T, vocab] (float64) of a whole sequence; with ``return_layers`` also the stream after every layer."""
    W = {k: v.to(F) for k, v in W.items()}
    eps = cfg["norm"]["eps"]
    x = W["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    taps, shared = [], {}

    def sublayer(x, p, q, fn, shift):
        h = rms_norm(x, 1 + W[p + "norm" + q], eps)
        y = fn(token_shift(h, W[p + "shift"]) if shift else h)
        y = y * torch.sigmoid(h @ W[p + "rg" + q].T + W[p + "rg" + q + ".b"])
        return x + rms_norm(y, 1 + W[p + "norm" + q + "b"], eps)
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        mix = {"parallel": lambda h: parallel(h, W, p + "mix.", m, eps),
               "attention": lambda h: conv_attention(h, W, p + "mix.", m, eps, shared),
               "attention_2": lambda h: window_attention(h, W, p + "mix.", m, eps, shared)}[L["type"]]
        x = sublayer(x, p, "1", mix, True)
        mlp = L.get("mlp")
        if mlp is not None:
            ff = (lambda h: clamped_ff(h, W, p + "mlp.", mlp["limit"])) if mlp["kind"] == "dense" else \
                (lambda h: routed_ff(h, W, p + "mlp.", mlp))
            x = sublayer(x, p, "2", ff, False)
        taps.append(x)
    logits = rms_norm(x, 1 + W["final.norm"], eps) @ W["embed"].T * cfg["logit_scale"]
    cap = cfg["logit_softcap"]
    logits = cap * torch.tanh(logits / cap)
    return (logits, taps) if return_layers else logits


def random_weights(cfg, seed=0):
    """bf16 tensors under the checkpoint's names: matrices N(0, 1 / fan_in) (queries and keys larger, so that the
    softmax is not flat), offset norm weights far from zero, shifts over (0, 1), router biases that matter."""
    gen = torch.Generator().manual_seed(seed)
    d, V = cfg["width"], cfg["vocab"]
    W = {}

    def mat(n, k, s=1.0):
        return (torch.randn(n, k, generator=gen) * s * k ** -0.5).to(torch.bfloat16)

    def vec(n, mean=0.0, s=0.1):
        return (mean + s * torch.randn(n, generator=gen)).to(torch.bfloat16)
    W["embed"] = mat(V, d, d ** 0.5)
    first = True
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        for q in ("1", "2") if L.get("mlp") is not None else ("1",):
            W[p + "norm" + q], W[p + "norm" + q + "b"] = vec(d, s=0.3), vec(d, s=0.3)
            W[p + "rg" + q], W[p + "rg" + q + ".b"] = mat(d, d, 2.0), vec(d, 0.3, 0.5)
        W[p + "shift"] = torch.rand(d, generator=gen).to(torch.bfloat16)
        x = p + "mix."
        if L["type"] == "parallel":
            l, r = m["left"], m["right"]
            H, G, D, Dv = l["heads"], l["kv_heads"], l["dim"], l["vdim"]
            W[x + "left.q"], W[x + "left.k"] = mat(H * D, d, 2.0), mat(G * D, d, 2.0)
            W[x + "left.v"], W[x + "left.o"] = mat(G * Dv, d), mat(d, H * Dv)
            H, D, Dv = r["heads"], r["dim"], r["vdim"]
            W[x + "right.q"], W[x + "right.k"], W[x + "right.v"] = mat(H * D, d), mat(H * D, d), mat(H * Dv, d)
            W[x + "right.g"], W[x + "right.o"] = mat(H * Dv, d, 2.0), mat(d, H * Dv)
            W[x + "right.norm"] = vec(H * Dv, 1.0, 0.3)
        else:
            H, G, D, Dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
            W[x + "q"], W[x + "k"], W[x + "v"], W[x + "o"] = mat(H * D, d), mat(G * D, d), mat(G * Dv, d), mat(d, H * Dv)
            if L["type"] == "attention":
                W[x + "q.norm"], W[x + "k.norm"] = vec(H * D, 1.5, 0.3), vec(G * D, 1.5, 0.3)
                for n, c in (("q", H * D), ("k", G * D), ("v", G * Dv)):
                    W[x + n + ".conv"] = (torch.randn(c, m["conv"], generator=gen) * 0.6).to(torch.bfloat16)
                W[x + "sink"], W[x + "g"] = vec(H, 0.5, 1.0), mat(H, d, 2.0)
            else:
                W[x + "q.norm"], W[x + "k.norm"] = vec(D, 1.5, 0.3), vec(D, 1.5, 0.3)
                W[x + "q.b"], W[x + "k.b"], W[x + "v.b"] = vec(H * D, s=0.3), vec(G * D, s=0.3), vec(G * Dv, s=0.3)
                W[x + "o.b"] = vec(d, s=0.2)
            if m.get("v_mix"):
                W[x + "vmix"] = torch.tensor(0.9 if first else 0.2 + 0.3 * float(torch.rand((), generator=gen))).to(torch.bfloat16)
                first = False
        mlp = L.get("mlp")
        f = p + "mlp."
        if mlp is not None and mlp["kind"] == "dense":
            n = mlp["ff"]
            W[f + "gate"], W[f + "up"], W[f + "down"] = mat(n, d, 1.5), mat(n, d, 1.5), mat(d, n)
        elif mlp is not None:
            n, E = mlp["expert"]["ff"], mlp["router"]["experts"]
            for e in range(E):
                W[f + f"e{e}.gate"], W[f + f"e{e}.up"], W[f + f"e{e}.down"] = mat(n, d, 1.5), mat(n, d, 1.5), mat(d, n)
            W[f + "router"], W[f + "router.b"] = mat(E, d, 2.0), vec(E, s=1.0)
    W["final.norm"] = vec(d, s=0.3)
    return W
