"""Plain float64 oracle of the Zifisun design: whole sequences, no cache, no batching, one function
per mechanism, every loop over tokens written out.  Shares no code with the product path.

A model is (config dict, weights dict name -> tensor).  ``forward`` returns the logits of every
position of one sequence and, optionally, the sum of the residual streams after every layer run.
"""
from __future__ import annotations

import math

import torch

F64 = torch.float64


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


def rms_norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


def softmax(s):
    e = torch.exp(s - s.max())
    return e / e.sum()


# ------------------------------------------------------------------ residual streams

def read_streams(xs, a):
    """xs [n, T, d] -> the sublayer's input [T, d] before its norm."""
    u = torch.zeros_like(xs[0])
    for s in range(xs.shape[0]):
        u = u + a[s] * xs[s]
    return u


def write_streams(xs, mix, out, y):
    """Every stream t becomes sum over s of mix[s, t] xs[s], plus out[t] y."""
    new = []
    for t in range(xs.shape[0]):
        v = out[t] * y
        for s in range(xs.shape[0]):
            v = v + mix[s, t] * xs[s]
        new.append(v)
    return torch.stack(new)


# ------------------------------------------------------------------ attention

def rotate_pairs(x, pos: int, base: float):
    """x [..., n]: entries 2i and 2i + 1 turn together by pos * base^(-2i/n)."""
    y = x.clone()
    n = x.shape[-1]
    for i in range(n // 2):
        ang = pos * base ** (-2.0 * i / n)
        c, s = math.cos(ang), math.sin(ang)
        y[..., 2 * i] = x[..., 2 * i] * c - x[..., 2 * i + 1] * s
        y[..., 2 * i + 1] = x[..., 2 * i + 1] * c + x[..., 2 * i] * s
    return y


def visible(i: int, size: int, first: int = 0) -> list:
    """The positions that position i sees: the last ``size`` (0: all) and those below ``first``."""
    return [j for j in range(i + 1) if not size or i - j < size or j < first]


def attend(q, k, v, scale: float, size: int, first: int = 0):
    """q [T, H, dk], k [T, G, dk], v [T, G, dv] -> [T, H, dv]."""
    T, H, _ = q.shape
    G, dv = k.shape[1], v.shape[2]
    out = torch.zeros(T, H, dv, dtype=F64)
    for i in range(T):
        js = visible(i, size, first)
        for h in range(H):
            g = h // (H // G)
            out[i, h] = softmax((k[js, g] @ q[i, h]) * scale) @ v[js, g]
    return out


def head_gate(o, h, wg):
    """o [T, H, dv]: every head times its own number sigmoid(wg h)[head]."""
    return o * sigmoid(h @ wg.T).unsqueeze(-1)


def attention(h, w: dict, pre: str, m: dict, eps: float):
    T = h.shape[0]
    H, G, dk, dv = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    mask = m.get("mask") or {}
    q = rms_norm((h @ w[pre + "q"].T).view(T, H, dk), w[pre + "q.norm"], eps)
    k = rms_norm((h @ w[pre + "k"].T).view(T, G, dk), w[pre + "k.norm"], eps)
    v = (h @ w[pre + "v"].T).view(T, G, dv)
    o = attend(q, k, v, float(m["scale"]), int(mask.get("size", 0)), int(mask.get("keep_first", 0)))
    return head_gate(o, h, w[pre + "g"]).reshape(T, H * dv) @ w[pre + "o"].T


def latent_attention(h, w: dict, pre: str, m: dict, eps: float):
    """Every head's keys and values written out."""
    T = h.shape[0]
    H, dn, dr, dv, R = int(m["heads"]), int(m["dim"]), int(m["rot_dim"]), int(m["vdim"]), int(m["kv_rank"])
    base = float(m["rot"]["base"])
    q = (rms_norm(h @ w[pre + "dq"].T, w[pre + "dq.norm"], eps) @ w[pre + "uq"].T).view(T, H, dn + dr)
    down = h @ w[pre + "dkv"].T
    c, kr = rms_norm(down[:, :R], w[pre + "dkv.norm"], eps), down[:, R:]
    q = torch.stack([torch.cat([q[t, :, :dn], rotate_pairs(q[t, :, dn:], t, base)], -1) for t in range(T)])
    kr = torch.stack([rotate_pairs(kr[t], t, base) for t in range(T)])
    k = torch.cat([(c @ w[pre + "uk"].T).view(T, H, dn), kr.view(T, 1, dr).expand(T, H, dr)], -1)
    v = (c @ w[pre + "uv"].T).view(T, H, dv)
    o = attend(q, k, v, float(m["scale"]), int((m.get("mask") or {}).get("size", 0)))
    return head_gate(o, h, w[pre + "g"]).reshape(T, H * dv) @ w[pre + "o"].T


# ------------------------------------------------------------------ feed-forward

def expert(h, up, down):
    return torch.relu(h @ up.T) ** 2 @ down.T


def route(s, corr, top: int, count: int, keep: int) -> list:
    """Indices chosen from one token's scores ``s`` [n]: by s + corr, within the ``keep`` best of
    ``count`` groups of neighbours (a group is as good as its best member)."""
    choice = s + corr
    per = len(s) // count
    groups = sorted(range(count), key=lambda g: -float(choice[g * per:(g + 1) * per].max()))[:keep]
    able = [e for e in range(len(s)) if e // per in groups]
    return sorted(able, key=lambda e: -float(choice[e]))[:top]


def experts_ff(h, w: dict, pre: str, m: dict):
    r = m["router"]
    E, K, ident = int(r["experts"]), int(r["top"]), int(r.get("identity") or 0)
    gr = r.get("groups") or {"count": 1, "keep": 1}
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        s = softmax(w[pre + "router"] @ h[t])
        assert len(s) == E + ident
        for e in route(s, w[pre + "correction"], K, int(gr["count"]), int(gr["keep"])):
            out[t] += s[e] * (h[t] if e >= E else expert(h[t], w[f"{pre}e{e}.up"], w[f"{pre}e{e}.down"]))
    if m.get("shared"):
        out = out + expert(h, w[pre + "shared.up"], w[pre + "shared.down"])
    return out


# ------------------------------------------------------------------ the model

def run_order(cfg: dict) -> list:
    n, lp = len(cfg["layers"]), cfg.get("loop")
    if not lp:
        return list(range(n))
    a, b = int(lp["start"]), int(lp["stop"])
    return list(range(a)) + list(range(a, b)) * int(lp["times"]) + list(range(b, n))


def forward(cfg: dict, weights: dict, tokens, layers_out: list | None = None) -> torch.Tensor:
    """Logits [T, vocab] (float64) of one sequence."""
    w = {k: v.to(F64) for k, v in weights.items()}
    eps = float(cfg["norm"]["eps"])
    x = w["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    xs = torch.stack([x] * int(cfg["streams"]))
    for i in run_order(cfg):
        L, p = cfg["layers"][i], f"l{i}."
        mixer = {"attention": attention, "latent_attention": latent_attention}[L["type"]]
        h = rms_norm(read_streams(xs, w[p + "hc1.in"]), w[p + "norm1"], eps)
        xs = write_streams(xs, w[p + "hc1.mix"], w[p + "hc1.out"], mixer(h, w, p + "mix.", L["mixer"], eps))
        if L.get("mlp"):
            h = rms_norm(read_streams(xs, w[p + "hc2.in"]), w[p + "norm2"], eps)
            xs = write_streams(xs, w[p + "hc2.mix"], w[p + "hc2.out"], experts_ff(h, w, p + "mlp.", L["mlp"]))
        if layers_out is not None:
            layers_out.append(xs.sum(0))
    return rms_norm(xs.sum(0), w["final.norm"], eps) @ w["head"].T


def layers_of(cfg: dict, weights: dict, tokens) -> torch.Tensor:
    """The sum of the streams after every layer run, [layer runs, T, width]."""
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
    """Random tensors of a config's shapes (values a bf16 checkpoint could hold), by name."""
    g = torch.Generator().manual_seed(seed)
    d, V, S = cfg["width"], cfg["vocab"], int(cfg["streams"])

    def rnd(*shape, std=1.0, mean=0.0):
        return (torch.randn(*shape, generator=g) * std + mean).to(torch.bfloat16).float()

    w = {"embed": rnd(V, d, std=0.8), "head": rnd(V, d, std=2 * d ** -0.5), "final.norm": rnd(d, std=0.1, mean=1.0)}

    def streams(name):
        w[name + ".in"], w[name + ".out"] = rnd(S, std=0.4, mean=1.0 / S), rnd(S, std=0.5, mean=0.7)
        w[name + ".mix"] = (0.8 * torch.eye(S) + rnd(S, S, std=0.3 / S)).to(torch.bfloat16).float()

    for i, spec in enumerate(cfg["layers"]):
        L, P, m = f"l{i}.", f"l{i}.mix.", spec["mixer"]
        H, dv = m["heads"], m["vdim"]
        w[L + "norm1"] = rnd(d, std=0.1, mean=1.0)
        streams(L + "hc1")
        if spec["type"] == "attention":
            G, dk = m["kv_heads"], m["dim"]
            w[P + "q"], w[P + "k"] = rnd(H * dk, d, std=d ** -0.5), rnd(G * dk, d, std=d ** -0.5)
            w[P + "v"] = rnd(G * dv, d, std=d ** -0.5)
            w[P + "q.norm"], w[P + "k.norm"] = rnd(dk, std=0.2, mean=1.3), rnd(dk, std=0.2, mean=1.0)
        else:
            dn, dr, Q, R = m["dim"], m["rot_dim"], m["q_rank"], m["kv_rank"]
            w[P + "dq"], w[P + "dq.norm"] = rnd(Q, d, std=d ** -0.5), rnd(Q, std=0.2, mean=1.2)
            w[P + "dkv"], w[P + "dkv.norm"] = rnd(R + dr, d, std=1.3 * d ** -0.5), rnd(R, std=0.2, mean=1.0)
            w[P + "uq"] = rnd(H * (dn + dr), Q, std=1.3 * Q ** -0.5)
            w[P + "uk"], w[P + "uv"] = rnd(H * dn, R, std=1.3 * R ** -0.5), rnd(H * dv, R, std=R ** -0.5)
        w[P + "g"], w[P + "o"] = rnd(H, d, std=2 * d ** -0.5), rnd(d, H * dv, std=(H * dv) ** -0.5)
        ml = spec.get("mlp")
        if ml:
            r = ml["router"]
            E, n = r["experts"], r["experts"] + int(r.get("identity") or 0)
            w[L + "norm2"] = rnd(d, std=0.1, mean=1.0)
            streams(L + "hc2")
            w[L + "mlp.router"], w[L + "mlp.correction"] = rnd(n, d, std=1.5 * d ** -0.5), rnd(n, std=0.15)
            forms = [(f"e{e}", ml["expert"]["ff"]) for e in range(E)]
            for name, f in forms + ([("shared", ml["shared"]["ff"])] if ml.get("shared") else []):
                w[f"{L}mlp.{name}.up"] = rnd(f, d, std=1.2 * d ** -0.5)
                w[f"{L}mlp.{name}.down"] = rnd(d, f, std=f ** -0.5)
    return w
