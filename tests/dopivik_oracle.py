"""Plain float64 oracle of the Dopivik design: whole sequences, no cache, no batching, one function
per mechanism, every loop over tokens written out.  Shares no code with the product path.

A model is (config dict, weights dict name -> tensor).  ``forward`` returns the logits of every
position of one sequence and, optionally, the residual stream after every layer.
"""
from __future__ import annotations

import math

import torch

F64 = torch.float64


def silu(z):
    return z / (1.0 + torch.exp(-z))


def softplus(z):
    return torch.where(z > 30.0, z, torch.log1p(torch.exp(torch.clamp(z, max=30.0))))


def rms(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def layer_norm(x, w, b, eps):
    mu = x.mean(-1, keepdim=True)
    var = ((x - mu) ** 2).mean(-1, keepdim=True)
    return (x - mu) / torch.sqrt(var + eps) * w + b


def rotate_half(x, pos: int, base: float, dims: int):
    """x [heads, dim]: entries i and i + dims/2 turn together by pos * base^(-2i/dims); entries from
    ``dims`` on pass."""
    y = x.clone()
    n = dims // 2
    for i in range(n):
        ang = pos * base ** (-2.0 * i / dims)
        c, s = math.cos(ang), math.sin(ang)
        y[:, i] = x[:, i] * c - x[:, i + n] * s
        y[:, i + n] = x[:, i + n] * c + x[:, i] * s
    return y


def chunked_attention(q, k, v, scale: float, cap: float, size: int):
    """q [T, H, dk], k [T, G, dk], v [T, G, dv] -> [T, H*dv]; position i sees j <= i of its own chunk of
    ``size`` positions (chunks start at multiples of ``size``); scores cap * tanh(q.k scale / cap)."""
    T, H, _ = q.shape
    G, dv = k.shape[1], v.shape[2]
    out = torch.zeros(T, H, dv, dtype=F64)
    for i in range(T):
        lo = (i // size) * size
        for h in range(H):
            g = h // (H // G)
            s = cap * torch.tanh((k[lo:i + 1, g] @ q[i, h]) * scale / cap)
            e = torch.exp(s - s.max())
            out[i, h] = (e / e.sum()) @ v[lo:i + 1, g]
    return out.reshape(T, H * dv)


def attention(h, w: dict, pre: str, m: dict):
    """The left mixer of a ``parallel`` layer."""
    T = h.shape[0]
    H, G, dk, dv = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    q = (h @ w[pre + "q"].T).view(T, H, dk)
    k = (h @ w[pre + "k"].T).view(T, G, dk)
    v = (h @ w[pre + "v"].T).view(T, G, dv)
    base, dims = float(m["rot"]["base"]), int(m["rot"]["dims"])
    q = torch.stack([rotate_half(q[t], t, base, dims) for t in range(T)])
    k = torch.stack([rotate_half(k[t], t, base, dims) for t in range(T)])
    o = chunked_attention(q, k, v, float(m["scale"]), float(m["softcap"]), int(m["mask"]["size"]))
    return (o * torch.sigmoid(h @ w[pre + "g"].T)) @ w[pre + "o"].T


def causal_conv(x, cw, b=None):
    """x [T, C], cw [C, taps] (last column: the current token), b [C]; zeros before the start."""
    T = x.shape[0]
    taps = cw.shape[1]
    y = torch.zeros_like(x)
    for t in range(T):
        for j in range(taps):
            s = t - (taps - 1 - j)
            if s >= 0:
                y[t] += cw[:, j] * x[s]
    return y + b if b is not None else y


def gated_delta(h, w: dict, pre: str, m: dict, eps: float):
    """The right mixer of a ``parallel`` layer: the delta rule with one decay per head."""
    T = h.shape[0]
    H, Gk, dk, dv = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    q = silu(causal_conv(h @ w[pre + "q"].T, w[pre + "q.conv"])).view(T, Gk, dk)
    k = silu(causal_conv(h @ w[pre + "k"].T, w[pre + "k.conv"])).view(T, Gk, dk)
    v = silu(causal_conv(h @ w[pre + "v"].T, w[pre + "v.conv"])).view(T, H, dv)
    q = q / torch.sqrt((q * q).sum(-1, keepdim=True) + 1e-6) * dk ** -0.5
    k = k / torch.sqrt((k * k).sum(-1, keepdim=True) + 1e-6)
    beta = torch.sigmoid(h @ w[pre + "b"].T)
    g = torch.exp(-torch.exp(w[pre + "A_log"]) * softplus(h @ w[pre + "a"].T + w[pre + "dt_bias"]))  # [T, H]
    out = torch.zeros(T, H, dv, dtype=F64)
    for hh in range(H):
        kk, qq = k[:, hh // (H // Gk)], q[:, hh // (H // Gk)]
        S = torch.zeros(dk, dv, dtype=F64)
        for t in range(T):
            S = g[t, hh] * S
            u = beta[t, hh] * (v[t, hh] - S.T @ kk[t])
            S = S + torch.outer(kk[t], u)
            out[t, hh] = S.T @ qq[t]
    out = rms(out, eps) * w[pre + "norm"] * silu(h @ w[pre + "g"].T).view(T, H, dv)
    return out.reshape(T, H * dv) @ w[pre + "o"].T


def parallel(h, w: dict, pre: str, m: dict, eps: float):
    a = attention(h, w, pre + "left.", m["left"])
    b = gated_delta(h, w, pre + "right.", m["right"], eps)
    return 0.5 * (rms(a, eps) * w[pre + "left.out"] + rms(b, eps) * w[pre + "right.out"])


def selective_scan(x, dt, A, B, C, D):
    """x, dt [T, c]; A [c, n]; B, C [T, n]; D [c]: S <- exp(dt A) S + dt x B;  y = S C + D x."""
    S = torch.zeros_like(A)
    y = torch.zeros_like(x)
    for t in range(x.shape[0]):
        S = torch.exp(dt[t].view(-1, 1) * A) * S + (dt[t] * x[t]).view(-1, 1) * B[t].view(1, -1)
        y[t] = S @ C[t] + D * x[t]
    return y


def mamba1(h, w: dict, pre: str, m: dict):
    inner, r, n = int(m["inner"]), int(m["dt_rank"]), int(m["state"])
    p = h @ w[pre + "in"].T
    x, z = p[:, :inner], p[:, inner:]
    x = silu(causal_conv(x, w[pre + "conv"], w[pre + "conv.b"]))
    q = x @ w[pre + "x"].T
    dt = softplus(q[:, :r] @ w[pre + "dt"].T + w[pre + "dt.b"])
    y = selective_scan(x, dt, -torch.exp(w[pre + "A_log"]), q[:, r:r + n], q[:, r + n:], w[pre + "D"])
    return (y * silu(z)) @ w[pre + "o"].T


def wkv_scan(r, k, v, dec, u):
    """r, k, dec [T, H, d], v [T, H, d], u [H, d]: o = (S + diag(u) k v^T)^T r;  S <- diag(dec) S + k v^T."""
    T, H, d = r.shape
    out = torch.zeros(T, H, d, dtype=r.dtype)
    for h in range(H):
        S = torch.zeros(d, d, dtype=r.dtype)
        for t in range(T):
            kv = torch.outer(k[t, h], v[t, h])
            out[t, h] = (S + u[h].view(d, 1) * kv).T @ r[t, h]
            S = dec[t, h].view(d, 1) * S + kv
    return out


def wkv(h, w: dict, pre: str, m: dict, eps: float):
    T = h.shape[0]
    H, d = int(m["heads"]), int(m["dim"])
    prev = torch.cat([torch.zeros_like(h[:1]), h[:-1]])
    mix = {s: h + (prev - h) * w[pre + "mu." + s] for s in "rkvgw"}
    r, k, v = ((mix[s] @ w[pre + s].T).view(T, H, d) for s in "rkv")
    gate = silu(mix["g"] @ w[pre + "g"].T)
    dec = torch.exp(-torch.exp(torch.tanh(mix["w"] @ w[pre + "w1"].T) @ w[pre + "w2"].T + w[pre + "w0"])).view(T, H, d)
    o = rms(wkv_scan(r, k, v, dec, w[pre + "u"]), eps).reshape(T, H * d)
    return (o * w[pre + "norm"] * gate) @ w[pre + "o"].T


def dense_ff(h, w: dict, pre: str):
    return torch.relu(h @ w[pre + "up"].T) ** 2 @ w[pre + "down"].T


def owner(cfg: dict, i: int) -> int:
    """The layer whose tensors layer i uses."""
    while cfg["layers"][i].get("weights_of") is not None:
        i = int(cfg["layers"][i]["weights_of"])
    return i


def forward(cfg: dict, weights: dict, tokens, layers_out: list | None = None) -> torch.Tensor:
    """Logits [T, vocab] (float64) of one sequence."""
    w = {k: v.to(F64) if v.is_floating_point() else v for k, v in weights.items()}
    eps = float(cfg["norm"]["eps"])
    tok = torch.as_tensor(tokens, dtype=torch.long)
    x = w["embed"][tok] * float(cfg["embedding"]["scale"])

    def ln(name, y):
        return layer_norm(y, w[name], w[name + ".b"], eps)

    for i, L in enumerate(cfg["layers"]):
        p = f"l{owner(cfg, i)}."
        m = L["mixer"]
        h = ln(p + "norm1", x)
        if L["type"] == "parallel":
            y = parallel(h, w, p + "mix.", m, eps)
        elif L["type"] == "mamba1":
            y = mamba1(h, w, p + "mix.", m)
        elif L["type"] == "wkv":
            y = wkv(h, w, p + "mix.", m, eps)
        else:
            raise ValueError(L["type"])
        x = x + ln(p + "norm1b", y)
        if L.get("mlp") is not None:
            x = x + ln(p + "norm2b", dense_ff(ln(p + "norm2", x), w, p + "mlp."))
        if layers_out is not None:
            layers_out.append(x.clone())
    return ln("final.norm", x) @ w["head"].T


def layers_of(cfg: dict, weights: dict, tokens) -> torch.Tensor:
    """The residual stream after every layer, [layers, T, width]."""
    out: list = []
    forward(cfg, weights, tokens, layers_out=out)
    return torch.stack(out)


def greedy(cfg: dict, w: dict, prompt, n: int) -> list:
    """``n`` tokens by repeated whole-sequence forwards, each the argmax of the last logits."""
    seq, out = list(prompt), []
    for _ in range(n):
        t = int(torch.argmax(forward(cfg, w, seq)[-1]))
        out.append(t)
        seq.append(t)
    return out


def random_weights(cfg: dict, seed: int = 0) -> dict:
    """Random tensors of a config's shapes (values a bf16 checkpoint could hold), by name.  The inner
    size of a wkv layer's two-stage decay is the mixer's ``w_rank`` (absent: 5)."""
    g = torch.Generator().manual_seed(seed)
    d, V = cfg["width"], cfg["vocab"]

    def rnd(*shape, std=1.0, mean=0.0):
        return (torch.randn(*shape, generator=g) * std + mean).to(torch.bfloat16).float()

    w = {"embed": rnd(V, d, std=0.8 / float(cfg["embedding"]["scale"])), "head": rnd(V, d, std=2 * d ** -0.5)}

    def norm(name):
        w[name], w[name + ".b"] = rnd(d, std=0.1, mean=1.0), rnd(d, std=0.1)

    norm("final.norm")
    for i, spec in enumerate(cfg["layers"]):
        if spec.get("weights_of") is not None:
            continue
        L, m, P = f"l{i}.", spec["mixer"], f"l{i}.mix."
        norm(L + "norm1")
        norm(L + "norm1b")
        if spec["type"] == "parallel":
            a, b, P, Q = m["left"], m["right"], P + "left.", P + "right."
            H, G, dk, dv = a["heads"], a["kv_heads"], a["dim"], a["vdim"]
            w[P + "q"], w[P + "k"] = rnd(H * dk, d, std=1.5 * d ** -0.5), rnd(G * dk, d, std=1.5 * d ** -0.5)
            w[P + "v"], w[P + "g"] = rnd(G * dv, d, std=d ** -0.5), rnd(H * dv, d, std=d ** -0.5)
            w[P + "o"] = rnd(d, H * dv, std=(H * dv) ** -0.5)
            H, Gk, dk, dv, taps = b["heads"], b["kv_heads"], b["dim"], b["vdim"], b["conv"]
            for n, rows in (("q", Gk * dk), ("k", Gk * dk), ("v", H * dv)):
                w[Q + n], w[Q + n + ".conv"] = rnd(rows, d, std=1.5 * d ** -0.5), rnd(rows, taps, std=0.5)
            w[Q + "b"], w[Q + "a"] = rnd(H, d, std=2 * d ** -0.5), rnd(H, d, std=d ** -0.5)
            w[Q + "A_log"], w[Q + "dt_bias"] = rnd(H, std=0.6, mean=-0.5), rnd(H, std=0.7, mean=-1.0)
            w[Q + "norm"], w[Q + "g"] = rnd(dv, std=0.1, mean=1.0), rnd(H * dv, d, std=d ** -0.5)
            w[Q + "o"] = rnd(d, H * dv, std=(H * dv) ** -0.5)
            w[P + "out"], w[Q + "out"] = rnd(d, std=0.2, mean=1.0), rnd(d, std=0.2, mean=1.0)
        elif spec["type"] == "mamba1":
            c, r, n, taps = m["inner"], m["dt_rank"], m["state"], m["conv"]
            w[P + "in"] = rnd(2 * c, d, std=d ** -0.5)
            w[P + "conv"], w[P + "conv.b"] = rnd(c, taps, std=0.5), rnd(c, std=0.1)
            w[P + "x"], w[P + "dt"], w[P + "dt.b"] = rnd(r + 2 * n, c, std=2 * c ** -0.5), rnd(c, r, std=r ** -0.5), rnd(c, std=0.7, mean=-2.0)
            w[P + "A_log"], w[P + "D"] = rnd(c, n, std=0.7, mean=0.3), rnd(c, std=0.3, mean=1.0)
            w[P + "o"] = rnd(d, c, std=c ** -0.5)
        else:
            H, k = m["heads"], m["dim"]
            r = int(m.get("w_rank", 5))
            for s in "rkvgw":
                w[P + "mu." + s] = rnd(d, std=0.25, mean=0.5)
            for s in "rkvg":
                w[P + s] = rnd(H * k, d, std=1.2 * d ** -0.5)
            w[P + "w1"], w[P + "w2"], w[P + "w0"] = rnd(r, d, std=d ** -0.5), rnd(H * k, r, std=r ** -0.5), rnd(H * k, std=1.0, mean=-1.5)
            w[P + "u"], w[P + "norm"] = rnd(H, k, std=0.5, mean=0.3), rnd(H * k, std=0.1, mean=1.0)
            w[P + "o"] = rnd(d, H * k, std=(H * k) ** -0.5)
        ml = spec.get("mlp")
        if ml is not None:
            norm(L + "norm2")
            norm(L + "norm2b")
            f = ml["ff"]
            w[L + "mlp.up"], w[L + "mlp.down"] = rnd(f, d, std=1.3 * d ** -0.5), rnd(d, f, std=f ** -0.5)
    return w
