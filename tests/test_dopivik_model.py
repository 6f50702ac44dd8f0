"""The Dopivik layer-list design in the engine against the plain float64 oracle
(tests/dopivik_oracle.py): each mechanism alone (the selective scan, wkv time mixing, chunked attention
with capped scores and an output gate, the delta rule with one decay per head, the normed pair, norms
on both sides of a sublayer, squared-ReLU layers, layers that use another layer's tensors), prefill
against token-by-token decoding, prompt portions down to two tokens, unequal batches, pages and state
slots that are reused, keys just inside and outside a chunk and at page borders, tokens far back in a
recurrent state, the first tokens, long decoding, odd sizes and sizes of one, and greedy generation
through the engine and the trace command.

Runs on the CPU (the ops' torch forms); the ``gpu`` tests at the end run the same comparisons
through the HIP kernels."""
import copy
import json
import subprocess
import sys

import numpy as np
import pytest
import torch

import dopivik_oracle as O
from k8s_llm_monitor_amd.engine import EngineConfig, LLMEngine, SamplingParams
from k8s_llm_monitor_amd.models.config import get_config, hybrid_config_from_dict, hybrid_config_to_dict
from k8s_llm_monitor_amd.models.hybrid import state_dict
from k8s_llm_monitor_amd.models.registry import build_model, config_from_dir
from k8s_llm_monitor_amd.ops import hybrid as hops
from test_hybrid_model import ROOT, Rig, _save, close, toks
from test_levovik_model import _bf16_close, _row_err


# ------------------------------------------------------------------ small configurations

def att(heads=4, kv=2, dim=12, vdim=10, scale=0.3, cap=6.0, chunk=20, dims=8, base=100.0):
    return {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale, "softcap": cap, "mask": {"size": chunk},
            "rot": {"dims": dims, "base": base}}


def delta(heads=4, kv=2, dim=6, vdim=10, conv=3):
    return {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "conv": conv}


def par(left=None, right=None, mlp=None):
    return {"type": "parallel", "mixer": {"left": left or att(), "right": right or delta()}, "mlp": mlp}


def mamba(inner=44, state=6, conv=3, dt_rank=5, mlp=None):
    return {"type": "mamba1", "mixer": {"inner": inner, "state": state, "conv": conv, "dt_rank": dt_rank}, "mlp": mlp}


def wkv(heads=3, dim=8, w_rank=5, mlp=None):
    return {"type": "wkv", "mixer": {"heads": heads, "dim": dim, "w_rank": w_rank}, "mlp": mlp}


def dense(ff=36):
    return {"kind": "dense", "ff": ff}


def make_cfg(layers, width=40, vocab=61, eps=1e-5, embed=3.0, share=()):
    """``share``: after the given layers, one more per entry that uses that layer's tensors."""
    layers = list(layers) + [dict(copy.deepcopy(layers[j]), weights_of=j) for j in share]
    return {"architecture": "Dopivik", "vocab": vocab, "width": width, "layers": layers, "norm": {"eps": eps},
            "embedding": {"scale": embed}}


FULL = make_cfg([wkv(mlp=dense(28)), par(mlp=dense(20)), mamba(mlp=dense()), par(att(3, 1, 16, 6, 0.25, 9.0, 33, 4), delta(2, 2, 8, 12, 4)),
                 mamba(30, 9, 4, 3)], share=(1, 0, 4))


def rig_for(cfg, seed=0, w=None, **kw):
    return Rig(dict(cfg, max_positions=kw.pop("max_positions", 1024)), w=w if w is not None else O.random_weights(cfg, seed), **kw)


# ------------------------------------------------------------------ mechanisms alone

SINGLE = {
    "parallel": [par()],
    "ones": [par(att(1, 1, 2, 1, 1.0, dims=2, chunk=1), delta(1, 1, 1, 1, 1))],
    "mqa-two-rotating-five-taps": [par(att(6, 1, 10, 4, dims=2, chunk=16), delta(6, 1, 4, 3, 5))],
    "own-keys-wide-values": [par(att(3, 3, 6, 9, dims=6, chunk=17), delta(3, 3, 9, 5, 2))],
    "chunk-beyond-prompt-low-cap": [par(att(chunk=500, cap=0.7))],
    "mamba": [mamba()], "mamba-ones": [mamba(1, 1, 1, 1)], "mamba-many-states": [mamba(10, 70, 6, 12)], "mamba-rank-1": [mamba(24, 16, 4, 1)],
    "wkv": [wkv()], "wkv-ones": [wkv(1, 1, 1)], "wkv-wide": [wkv(1, 36, 7)], "wkv-many-heads": [wkv(7, 4, 3)],
    "dense": [mamba(mlp=dense())], "dense-ff1": [wkv(mlp=dense(1))], "dense-parallel": [par(mlp=dense(50))]}


@pytest.mark.parametrize("name", list(SINGLE))
def test_single_mechanism_whole_prompt(name):
    cfg = make_cfg(SINGLE[name])
    rig = rig_for(cfg, 3)
    t = toks(45, cfg["vocab"], 1)
    close(rig.run_cut("a", t, [45]), O.forward(cfg, rig.w, t))


ODD = make_cfg([par(att(5, 5, 7, 3, dims=6, chunk=11), delta(6, 3, 5, 7, 2), mlp=dense(11)), mamba(19, 5, 3, 7, mlp=dense(9)),
                wkv(3, 5, 2, mlp=dense(3)), par(att(2, 1, 11, 13, dims=10, chunk=7), delta(1, 1, 13, 3, 6))],
               width=37, vocab=53, share=(2, 0))


def test_odd_sizes_everywhere():
    """Widths, ranks and head sizes that are multiples of nothing (rotated sizes stay even)."""
    rig = rig_for(ODD, 31)
    t = toks(41, 53, 3)
    want = O.forward(ODD, rig.w, t)
    for cuts in ([41], [3, 2, 17], [1]):
        close(rig.run_cut("a", t, cuts), want)


def test_layer_outputs_match_oracle():
    rig = rig_for(FULL, 5)
    t = toks(19, FULL["vocab"], 3)
    rig.model.layer_probe = []
    rig.run_cut("a", t, [19])
    layers = O.layers_of(FULL, rig.w, t)
    assert len(rig.model.layer_probe) == layers.shape[0] == 8
    for got, want in zip(rig.model.layer_probe, layers):
        close(got, want)
    rig.model.layer_probe = None


def _i32(*a):
    return torch.tensor(a, dtype=torch.int32)


def test_ops_against_oracle_functions():
    g = torch.Generator().manual_seed(1)
    rnd = lambda *s: torch.randn(*s, generator=g)
    # a branch through its own layer norm into the stream, then the next norm; one result and a normed pair
    x, a, b = rnd(5, 12) * 2 + 1, rnd(5, 12) * 3 - 1, rnd(5, 12)
    p, q = (rnd(12), rnd(12)), (rnd(12), rnd(12))
    wa, wb = rnd(12), rnd(12)
    ln = lambda v, wb_: O.layer_norm(v, wb_[0].double(), wb_[1].double(), 1e-5)
    res = x.clone()
    h = hops.join_norm(res, (a,), p, q, 1e-5, torch.float32)
    want = x.double() + ln(a.double(), p)
    close(res, want, tol=1e-6)
    close(h, ln(want, q), tol=1e-6)
    res = x.clone()
    assert hops.join_norm(res, (a, b), p, None, 1e-5, torch.float32, branch_w=(wa, wb), mix=0.5) is None
    pair = 0.5 * (O.rms(a.double(), 1e-5) * wa.double() + O.rms(b.double(), 1e-5) * wb.double())
    close(res, x.double() + ln(pair, p), tol=1e-6)
    res = x.clone()
    close(hops.join_norm(res, (), None, q, 1e-5, torch.float32), ln(x.double(), q), tol=1e-6)
    assert torch.equal(res, x)
    # activations
    z = rnd(4, 9) * 3
    close(hops.activation(z, "relu_sq"), torch.relu(z.double()) ** 2, tol=1e-6)
    close(hops.activation(z, "tanh"), torch.tanh(z.double()), tol=1e-6)
    # mixes with the previous token: two segments, one that carries on and one that starts in a used slot
    hh, mu, st = rnd(7, 6), rnd(5, 6), rnd(3, 6)
    st0 = st.clone()
    got = hops.token_mix(hh, mu, st, _i32(0, 3, 7), _i32(4, 0), _i32(2, 0), torch.float32)
    for s, (lo, hi, first) in enumerate(((0, 3, st0[2]), (3, 7, torch.zeros(6)))):
        for t in range(lo, hi):
            prev = first if t == lo else hh[t - 1]
            for j in range(5):
                close(got[t, j], (hh[t] + (prev - hh[t]) * mu[j]).double(), tol=1e-6)
    assert torch.equal(st[2], hh[2]) and torch.equal(st[0], hh[6]) and torch.equal(st[1], st0[1])


def test_chunked_capped_attention_op():
    """Prompt portions and single decode rows over the pages against the written-out attention."""
    g = torch.Generator().manual_seed(4)
    H, G, dk, dv, n = 4, 2, 6, 5, 40
    qkv = torch.randn(n, H * dk + G * dk + G * dv, generator=g) * 1.5
    q, k = qkv[:, :H * dk].double().view(n, H, dk), qkv[:, H * dk:H * dk + G * dk].double().view(n, G, dk)
    v = qkv[:, H * dk + G * dk:].double().view(n, G, dv)
    kc, vc = torch.zeros(4, 16, G * dk), torch.zeros(4, G, dv, 16)
    order = [2, 0, 3]  # the sequence's pages
    bt = _i32(*order).view(1, 3)
    for t in range(n):
        kc[order[t // 16], t % 16] = k[t].float().reshape(-1)
        vc[order[t // 16], :, :, t % 16] = v[t].float()
    for size, cap in ((1, 5.0), (7, 2.0), (16, 1.0), (17, 3.0), (40, 0.5), (100, 4.0)):
        want = O.chunked_attention(q, k, v, 0.4, cap, size)
        kw = dict(chunked=True, cap=cap)
        for a, b in ((0, 40), (5, 7), (15, 34)):
            got = hops.window_attention_prefill(qkv[a:b].contiguous(), kc, vc, _i32(0, b - a), _i32(a), bt, H, G, dk, dv, 0.4, size, False, **kw)
            close(got, want[a:b], tol=1e-5)
        for t in (0, 6, 7, 15, 16, 33, 34, 39):
            got = hops.window_attention_decode(qkv[t:t + 1], kc, vc, bt, _i32(t + 1), H, G, dk, dv, 0.4, size, False, **kw)
            close(got, want[t:t + 1], tol=1e-5)


def _delta_case(g, n, H, Gk, dk, dv):
    """Rows [q | k | v | beta | a] and the other inputs of the delta rule with one decay per head, and its
    outputs written out in float64."""
    qkv = torch.randn(n, 2 * Gk * dk + H * dv + 2 * H, generator=g)
    zb, a_log = torch.randn(H, generator=g), torch.randn(H, generator=g) * 0.5 - 0.5
    x = qkv.double()
    q, k = x[:, :Gk * dk].view(n, Gk, dk), x[:, Gk * dk:2 * Gk * dk].view(n, Gk, dk)
    c = 2 * Gk * dk + H * dv
    v, beta = x[:, 2 * Gk * dk:c].view(n, H, dv), torch.sigmoid(x[:, c:c + H])
    dec = torch.exp(-torch.exp(a_log.double()) * O.softplus(x[:, c + H:] + zb.double()))
    q = q / torch.sqrt((q * q).sum(-1, keepdim=True) + 1e-6) * dk ** -0.5
    k = k / torch.sqrt((k * k).sum(-1, keepdim=True) + 1e-6)
    out = torch.zeros(n, H, dv, dtype=torch.float64)
    for h in range(H):
        S = torch.zeros(dk, dv, dtype=torch.float64)
        for t in range(n):
            S = dec[t, h] * S
            S = S + torch.outer(k[t, h // (H // Gk)], beta[t, h] * (v[t, h] - S.T @ k[t, h // (H // Gk)]))
            out[t, h] = S.T @ q[t, h // (H // Gk)]
    kw = dict(a_log=a_log, beta_col=c, unit=True, z_col=c + H)
    return qkv, zb, kw, out.reshape(n, H * dv)


def _wkv_case(g, n, H, dk):
    rkv, z = torch.randn(n, 3 * H * dk, generator=g), torch.randn(n, H * dk, generator=g)
    w0, u = torch.randn(H * dk, generator=g) - 1.0, torch.randn(H, dk, generator=g)
    r, k, v = (rkv[:, i * H * dk:(i + 1) * H * dk].double().view(n, H, dk) for i in range(3))
    dec = torch.exp(-torch.exp(z.double() + w0.double())).view(n, H, dk)
    return rkv, z, w0, u, O.wkv_scan(r, k, v, dec, u.double()).reshape(n, H * dk)


def _scan_case(g, n, C, N, mean=-1.0):
    """Inputs of the selective scan (B, C behind 3 other columns) and its gated outputs in float64."""
    xc, q = torch.randn(n, C, generator=g), torch.randn(n, 3 + 2 * N, generator=g)
    dt, db = torch.randn(n, C, generator=g) + mean, torch.randn(C, generator=g) * 0.5
    al, D, pr = torch.randn(C, N, generator=g) * 0.7, torch.randn(C, generator=g), torch.randn(n, 2 * C, generator=g)
    y = O.selective_scan(xc.double(), O.softplus(dt.double() + db.double()), -torch.exp(al.double()), q[:, 3:3 + N].double(),
                         q[:, 3 + N:].double(), D.double())
    return (xc, q, dt, db, al, D, pr), y * O.silu(pr[:, C:].double())


def test_recurrences_across_segments():
    """Each recurrence over three segments of one sequence equals one pass; the slot holds leftovers of
    an earlier sequence, which a sequence that starts must not see."""
    g = torch.Generator().manual_seed(2)
    n = 21
    parts = ((0, 4), (4, 5), (5, 21))

    def run(state, fn):
        return torch.cat([fn(slice(a, b), (_i32(0, b - a), _i32(a), _i32(1))) for a, b in parts])

    qkv, zb, kw, want = _delta_case(g, n, 4, 2, 3, 5)
    st = torch.randn(3, 4, 5, 3, generator=g)
    close(run(st, lambda s, seg: hops.decay_scan(qkv[s], 0, 6, 12, qkv[s], zb, st, *seg, 4, 2, 3, 5, 3 ** -0.5, beta=qkv[s], **kw)), want,
          tol=1e-5)
    rkv, z, w0, u, want = _wkv_case(g, n, 3, 4)
    st2 = torch.randn(3, 3, 4, 4, generator=g)
    close(run(st2, lambda s, seg: hops.decay_scan(rkv[s], 0, 12, 24, z[s], w0, st2, *seg, 3, 3, 4, 4, 1.0, decay="exp_exp", bonus=u)), want,
          tol=1e-5)
    (xc, q, dt, db, al, D, pr), want = _scan_case(g, n, 6, 5)
    st3 = torch.randn(3, 6, 5, generator=g)
    close(run(st3, lambda s, seg: hops.selective_scan(xc[s], q[s], 3, 8, dt[s], db, al, D, pr[s], 6, st3, *seg)), want, tol=1e-5)


# ------------------------------------------------------------------ cuts, decoding, batches

def test_prefill_equals_token_by_token_and_portions():
    rig = rig_for(FULL, 6)
    t = toks(70, FULL["vocab"], 4)
    want = O.forward(FULL, rig.w, t)
    for cuts in ([70], [], [2, 2, 3, 16, 1, 31], [15, 17, 16, 2], [33, 2, 2, 2], [20, 20, 20]):
        close(rig.run_cut("a", t, cuts), want)


def test_first_tokens_and_single_token_prompt():
    """Shorter than the convolutions' taps and with no previous token: the zeros before the start."""
    rig = rig_for(FULL, 7)
    for n in (1, 2, 3):
        t = toks(n, FULL["vocab"], 10 + n)
        close(rig.run_cut("a", t, [n]), O.forward(FULL, rig.w, t))
        close(rig.run_cut("a", t, []), O.forward(FULL, rig.w, t))


def test_long_decoding_over_pages_and_chunks():
    rig = rig_for(FULL, 8)
    t = toks(150, FULL["vocab"], 5)
    close(rig.run_cut("a", t, [20]), O.forward(FULL, rig.w, t))  # 130 decode steps: 9 pages, 7 and 4 chunks


PLANS = (([("a", 17), ("b", 2), ("c", 3)], ["c"]), ([("a", 1), ("b", 19), ("d", 30)], ["b"]),
         ([("a", 1), ("d", 1), ("e", 16)], []), ([("a", 31), ("d", 2), ("e", 1)], ["a"]), ([("d", 1), ("e", 1)], []),
         ([("d", 3), ("e", 26)], ["d", "e"]))


def _run_plans(rig, T):
    got, at = {n: [] for n in T}, {n: 0 for n in T}
    for plan, end in PLANS:
        entries = []
        for n, k in plan:
            entries.append((n, T[n][at[n]:at[n] + k]))
            at[n] += k
        for n, lg in rig.step(entries, end).items():
            got[n].append(lg)
    assert not rig.live and all(at[n] == len(T[n]) for n in T)
    return {n: torch.cat(v) for n, v in got.items()}


def _plan_tokens(V):
    return {n: toks(k, V, s) for n, k, s in (("a", 50, 1), ("b", 21, 2), ("c", 3, 3), ("d", 37, 4), ("e", 44, 5))}


def test_unequal_batch_equals_each_alone_and_reuse():
    """Live requests with portions beside decode tokens; one ends and its pages and slot are taken by a
    new request whose logits must not see the old pages, states, convolution inputs or previous token."""
    rig = rig_for(FULL, 9, num_blocks=12)
    T = _plan_tokens(FULL["vocab"])
    got = _run_plans(rig, T)
    for n in T:
        close(got[n], O.forward(FULL, rig.w, T[n]))
    assert rig.blocks.num_free == 12 and len(rig.blocks._free_slots) == 4


# ------------------------------------------------------------------ shared tensors

def test_shared_tensors_have_their_own_state():
    """A layer that uses another's tensors equals the same model with a copy of them; the sharing may be
    a chain, may point forward, and adds no parameters."""
    base = [wkv(mlp=dense(12)), par(att(chunk=9)), mamba(mlp=dense(10))]
    cfg = make_cfg(base, share=(2, 1, 0))
    cfg["layers"].append(dict(copy.deepcopy(base[2]), weights_of=3))  # a chain: layer 3 uses layer 2's
    cfg["layers"].insert(0, dict(copy.deepcopy(base[2]), weights_of=3))  # points forward: layer 3 is the mamba layer now
    for i, L in enumerate(cfg["layers"][1:], 1):
        if "weights_of" in L:
            L["weights_of"] += 1
    w = O.random_weights(cfg, 4)
    t = toks(40, cfg["vocab"], 2)
    want = O.forward(cfg, w, t)
    plain = copy.deepcopy(cfg)
    w2 = dict(w)
    for i, L in enumerate(plain["layers"]):
        j = O.owner(cfg, i)
        L.pop("weights_of", None)
        w2.update({f"l{i}." + k[len(f"l{j}."):]: v for k, v in w.items() if k.startswith(f"l{j}.")})
    close(O.forward(plain, w2, t), want, tol=1e-12)
    a, b = rig_for(cfg, w=w), rig_for(plain, w=w2)
    for cuts in ([40], [7, 2, 20]):
        close(a.run_cut("a", t, cuts), want)
        close(b.run_cut("a", t, cuts), want)
    assert a.model.resident_weight_bytes() < b.model.resident_weight_bytes()
    assert sorted(state_dict(a.model)) == sorted(w)
    assert a.model.cache_bytes() == b.model.cache_bytes()
    assert a.runner.memory_report()["kv_cache_bytes"] > 0


# ------------------------------------------------------------------ faults made visible

def _spiked(cfg, seed, far, n, scale_up=(), by=4.0):
    """Weights and a prompt in which ONE position stands out: its token (the last id, which occurs nowhere
    else) has a large embedding, and the named projections are scaled up."""
    w = O.random_weights(cfg, seed)
    t = toks(n, cfg["vocab"] - 1, seed)
    special = cfg["vocab"] - 1
    t[far] = special
    w["embed"] = w["embed"].clone()
    w["embed"][special] *= 6.0
    for name in scale_up:
        w[name] = w[name] * by
    return w, t


def _moved(cfg, w, t, far):
    """The oracle's logits with another token at ``far``."""
    t2 = list(t)
    t2[far] = 0
    return O.forward(cfg, w, t2)


def _only(cfg, side):
    """A model of one ``parallel`` layer in which only one side reaches the stream."""
    def fix(w):
        other = {"left": "right", "right": "left"}[side]
        w[f"l0.mix.{other}.out"] = torch.zeros_like(w[f"l0.mix.{other}.out"])
        return w
    return fix


@pytest.mark.parametrize("chunk", [1, 2, 15, 16, 17, 24])
def test_chunk_edges(chunk):
    """A spiked key is seen by every later position of its chunk and by no position of the next, wherever
    the prompt is cut and whether those positions are prefilled or decoded."""
    cfg = make_cfg([par(att(2, 1, 8, 8, chunk=chunk, dims=4))], width=24, vocab=37)
    for far in sorted({chunk - 1, 2 * chunk - 1, chunk, 2 * chunk - min(2, chunk)}):
        n = far + chunk + 4
        w, t = _spiked(cfg, 11, far, n, ("l0.mix.left.v",))
        w = _only(cfg, "left")(w)
        want, other = O.forward(cfg, w, t), _moved(cfg, w, t, far)
        end = (far // chunk + 1) * chunk  # the first position that must not see it
        d = (want - other).abs().amax(-1)
        assert all(float(d[p]) > 1e-3 for p in range(far, end)) and all(float(d[p]) < 1e-12 for p in range(end, n))
        for cuts in ([n], [far], [far + 1], [end], [max(1, end - 1), 2], [2] * (n // 2 + 1)):
            close(rig_for(cfg, w=w).run_cut("a", t, cuts), want, tol=1e-4)


def test_far_key_in_a_long_chunk_with_a_peaked_score():
    """One key takes a large part of the softmax of every later query of its chunk, hundreds of tokens on
    (scores near the cap), and none of the next chunk."""
    cfg = make_cfg([par(att(2, 1, 8, 8, 1.0, 12.0, 320, dims=4, base=1e4))], width=24, vocab=37, embed=1.0)
    n, far = 330, 20
    w, t = _spiked(cfg, 13, far, n)
    w = _only(cfg, "left")(w)
    e = w["embed"]
    e[:, 0], e[:, 1], e[:, 2] = 1.0, 0.0, 0.0  # axis 0 - axis 2: the same for all; axis 1 - axis 2: the special token only
    e[36, 1] = 4.0
    w["l0.norm1"], w["l0.norm1.b"] = torch.ones(24), torch.zeros(24)
    eye = torch.eye(24)
    for h in range(2):  # the last entry of a head does not turn
        w["l0.mix.left.q"][h * 8 + 7] = 8.0 * (eye[0] - eye[2])
    w["l0.mix.left.k"][7] = 8.0 * (eye[1] - eye[2])
    want = O.forward(cfg, w, t)
    d = (want - _moved(cfg, w, t, far)).abs().amax(-1)
    assert float(d[319]) > 0.1 and float(d[320]) < 1e-12
    for cuts in ([n], [310], [100, 2, 64, 130], [far + 12]):
        close(rig_for(cfg, w=w, num_blocks=32).run_cut("a", t, cuts), want, tol=1e-4)


def _slow_state(kind):
    """A one-layer model whose recurrent state forgets slowly, with a far spiked token."""
    layer = {"mamba": mamba(20, 4, 3, 3), "wkv": wkv(2, 6, 3), "delta": par(right=delta(2, 1, 6, 6, 3))}[kind]
    cfg = make_cfg([layer], width=24, vocab=37)
    n, far = 330, 20
    w, t = _spiked(cfg, 14, far, n)
    if kind == "mamba":  # small steps, slow decays; the special token alone takes a large step (x column up)
        w["l0.mix.dt.b"] = torch.full((20,), -6.0)
        w["l0.mix.A_log"] = torch.full((20, 4), -1.0)
        w["l0.mix.D"] = torch.zeros(20)
        e = w["embed"]
        e[:, 0], e[:, 1] = 0.0, 1.0
        e[36, 0] = 8.0
        w["l0.norm1"], w["l0.norm1.b"] = torch.ones(24), torch.zeros(24)
        eye = torch.eye(24)
        w["l0.mix.in"][0] = 3.0 * eye[0]  # channel 0: the marker
        w["l0.mix.conv"][0], w["l0.mix.conv.b"][0] = torch.tensor([0.0, 0.0, 1.0]), 0.0
        w["l0.mix.x"][:3] = 0.0
        w["l0.mix.x"][0, 0] = 1.0
        w["l0.mix.dt"] = torch.zeros(20, 3)
        w["l0.mix.dt"][:, 0] = 0.5
    elif kind == "wkv":
        w["l0.mix.w0"] = torch.full((12,), -7.0)
        w["l0.mix.w2"] = w["l0.mix.w2"] * 0.1
        w["l0.mix.k"] = w["l0.mix.k"] * 0.3
    else:
        w = _only(cfg, "right")(w)
        w["l0.mix.right.A_log"], w["l0.mix.right.dt_bias"] = torch.full((2,), -5.0), torch.full((2,), -4.0)
        e = w["embed"]
        e[:, 0], e[:, 1], e[:, 2] = 1.0, 0.0, 0.0
        e[36, 1] = 2.0
        w["l0.norm1"], w["l0.norm1.b"] = torch.ones(24), torch.zeros(24)
        eye = torch.eye(24)
        w["l0.mix.right.q"][0], w["l0.mix.right.k"][0] = 3.0 * (eye[0] - eye[2]), 3.0 * (eye[1] - eye[2])
        for nme in ("q", "k", "v"):  # the current token's tap dominates
            w[f"l0.mix.right.{nme}.conv"][:, -1] = 1.5
    return cfg, w, t, far, n


@pytest.mark.parametrize("kind", ["mamba", "wkv", "delta"])
def test_far_token_in_the_recurrent_state(kind):
    """A state lost at the start of a portion or of a decode step, or a slot mixed up, would show."""
    cfg, w, t, far, n = _slow_state(kind)
    want = O.forward(cfg, w, t)
    assert float((want[n - 1] - _moved(cfg, w, t, far)[n - 1]).abs().max()) > 0.02
    for cuts in ([n], [310], [100, 2, 64, 130], [far + 12]):
        close(rig_for(cfg, w=w, num_blocks=32).run_cut("a", t, cuts), want, tol=1e-4)


@pytest.mark.parametrize("kind", ["mamba", "wkv", "delta"])
def test_inputs_of_earlier_tokens_cross_portions(kind):
    """A portion that starts right after the spiked token still convolves it, or mixes it in as the previous
    token: with that part of the state lost, the next positions would move."""
    layer, name, by = {"mamba": (mamba(20, 4, 5, 3), "l0.mix.conv", 3.0), "wkv": (wkv(2, 6, 3), "l0.mix.mu.v", 1.5),
                       "delta": (par(right=delta(2, 2, 6, 6, 5)), "l0.mix.right.v.conv", 4.0)}[kind]
    cfg = make_cfg([layer], width=24, vocab=37)
    far = 16
    w, t = _spiked(cfg, 12, far, far + 8, (name,), by)
    want = O.forward(cfg, w, t)
    d = (want - _moved(cfg, w, t, far)).abs().amax(-1)
    assert float(d[far - 1]) < 1e-12 and float(d[far + 1]) > 1e-2  # causal, and the next token depends on it
    for cuts in ([far + 1], [far + 1, 2, 2], [far, 1, 1, 2], [far + 3], [2] * 12):
        close(rig_for(cfg, w=w).run_cut("a", t, cuts), want, tol=1e-4)


def test_every_tensor_and_constant_matters_and_is_read():
    """The oracle moves when any tensor or constant is changed, and the engine follows it."""
    cfg = make_cfg([par(att(3, 1, 8, 6, dims=4, chunk=5, cap=1.5), mlp=dense(12)), mamba(14, 4, 3, 3), wkv(2, 6, 3)], width=24, vocab=37)
    w = O.random_weights(cfg, 16)
    t = toks(14, 37, 6)
    want = O.forward(cfg, w, t)
    g = torch.Generator().manual_seed(3)
    for name, v in w.items():
        w0 = dict(w)
        w0[name] = v + 0.5 * v.abs().mean() * torch.randn(v.shape, generator=g)
        assert float((O.forward(cfg, w0, t) - want).abs().max()) > 1e-4, name
    variants = []
    for path, val in ((("embedding", "scale"), 1.0), (("layers", 0, "mixer", "left", "scale"), 1.0), (("layers", 0, "mixer", "left", "softcap"), 50.0),
                      (("layers", 0, "mixer", "left", "mask", "size"), 6), (("layers", 0, "mixer", "left", "rot", "base"), 5.0),
                      (("layers", 0, "mixer", "left", "rot", "dims"), 8), (("norm", "eps"), 0.1)):
        c2 = copy.deepcopy(cfg)
        node = c2
        for k in path[:-1]:
            node = node[k]
        node[path[-1]] = val
        assert float((O.forward(c2, w, t) - want).abs().max()) > 1e-3, path
        variants.append(c2)
    for c in [cfg] + variants:
        ref = O.forward(c, w, t)
        for cuts in ([14], [3, 2]):
            close(rig_for(c, w=w).run_cut("a", t, cuts), ref, tol=1e-4)


def test_rotation_and_chunks_count_from_zero_on_any_pages():
    """Positions count from 0 in every sequence whatever pages and slots it gets; large positions keep
    their accuracy."""
    cfg = make_cfg([par(att(2, 2, 12, 8, 0.4, chunk=150, dims=12, base=20.0)), par(att(2, 1, 12, 8, 0.4, chunk=64, dims=8, base=20.0))],
                   width=24, vocab=37)
    rig = rig_for(cfg, 15, num_blocks=48)
    t = toks(420, 37, 9)
    want = O.forward(cfg, rig.w, t)
    rig.step([("z", toks(90, 37, 1))])  # holds the first pages and slot 0
    close(rig.run_cut("a", t, [200, 3, 200]), want, tol=5e-4)


# ------------------------------------------------------------------ engine entry points

def test_greedy_generation_through_engine(tmp_path):
    w = O.random_weights(FULL, 21)
    d = _save(tmp_path, FULL, w)
    assert config_from_dir(d).arch == "dopivik"
    eng = LLMEngine(EngineConfig(model=str(d), weights=str(d), max_num_seqs=3, max_model_len=256, num_blocks=40,
                                 dtype="float32", max_prefill_tokens=16, mixed_prefill_tokens=8), device="cpu")
    prompts = [toks(n, FULL["vocab"], 30 + n) for n in (4, 29, 18, 40)]  # 4 requests over 3 slots: one waits
    seqs = eng.generate(prompts, SamplingParams(max_tokens=10, temperature=0.0, ignore_eos=True))
    for p, s in zip(prompts, seqs):
        assert s.output_ids == O.greedy(FULL, w, p, 10)
    st = eng.stats()
    assert st["mixed_steps"] > 0 and st["kv_blocks_free"] == st["kv_blocks_total"]


def test_preset_round_trip_and_registry():
    c = get_config("dopivik-tiny")
    assert hybrid_config_from_dict(hybrid_config_to_dict(c), c.name) == c
    m = build_model(c, device="cpu", dtype=torch.float32)
    w = state_dict(m)
    assert w["l2.mix.w1"].shape == (8, c.d_model) and w["l1.mix.left.out"].shape == (c.d_model,) and "l2.norm2b" not in w
    assert not any(k.startswith(("l4.", "l5.", "l6.")) for k in w) and w["final.norm.b"].shape == (c.d_model,)
    cfg = hybrid_config_to_dict(c)
    eng = LLMEngine(EngineConfig(model="dopivik-tiny", max_num_seqs=2, max_model_len=128, num_blocks=16,
                                 dtype="float32"), device="cpu")
    p = toks(11, c.vocab_size, 1)
    s = eng.generate([p], SamplingParams(max_tokens=6, temperature=0.0, ignore_eos=True))[0]
    assert s.output_ids == O.greedy(cfg, w, p, 6)


def test_config_errors_are_loud():
    ok = O.random_weights(make_cfg([par()]), 1)
    for bad in (par(att(4, 3)), par(right=delta(4, 3)), par(att(dims=7)), par(att(dims=14)), mamba(0), dict(par(), type="parallel_2")):
        with pytest.raises(ValueError):
            rig_for(make_cfg([bad]), 1, w=ok)
    for share in ([par(), dict(par(att(chunk=9)), weights_of=0)], [dict(par(), weights_of=1), dict(par(), weights_of=0)],
                  [par(), dict(par(), weights_of=2)]):
        with pytest.raises(ValueError):
            rig_for(make_cfg(share), 1, w=ok)


def test_trace_command_replays_steps(tmp_path):
    """The command-line replayer: portions, a mixed step, a decode-only step, ends and reuse."""
    w = O.random_weights(FULL, 22)
    d = _save(tmp_path, FULL, w)
    V = FULL["vocab"]
    A, B = toks(23, V, 1), toks(9, V, 2)
    steps = [{"step": 0, "entries": [{"id": "x", "tokens": A[:20], "want": [0, 19]}], "end": []},
             {"step": 1, "entries": [{"id": "y", "tokens": B[:8], "want": [7]}, {"id": "x", "tokens": A[20:21], "want": [0]}],
              "end": []},
             {"step": 2, "entries": [{"id": "x", "tokens": A[21:22], "want": []}, {"id": "y", "tokens": B[8:], "want": [0]}],
              "end": ["y"]},
             {"step": 3, "entries": [{"id": "x", "tokens": A[22:], "want": [0]}], "end": ["x"]}]
    out = tmp_path / "o"
    r = subprocess.run([sys.executable, "-m", "k8s_llm_monitor_amd.cmd.trace_run", "--model", str(d), "--dtype", "float32",
                        "--out", str(out), "--max-tokens", "64", "--device", "cpu"],
                       input="\n".join(json.dumps(s) for s in steps) + "\n", capture_output=True, text=True, cwd=ROOT)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [ln for ln in r.stdout.splitlines() if ln.startswith("done")] == [f"done {i}" for i in range(4)]
    wa, wb = O.forward(FULL, w, A), O.forward(FULL, w, B)

    def rd(i):
        return torch.from_numpy(np.fromfile(out / f"{i}.f32", dtype="<f4").reshape(-1, V).copy())

    close(rd(0), wa[[0, 19]])
    close(rd(1), torch.stack([wb[7], wa[20]]))  # entry order, not the engine's row order
    close(rd(2), wb[8:9])
    close(rd(3), wa[22:23])


# ------------------------------------------------------------------ the same through the HIP kernels

def _bf16_ref_err(cfg, w, t, want, **kw):
    """What bf16 rounding alone costs on this model and prompt: the torch forms on the CPU, in bf16,
    against the oracle (row errors over the logits' scale)."""
    return _row_err(rig_for(cfg, w=w, dtype=torch.bfloat16, **kw).run_cut("a", t, [len(t)]), want)


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_gpu_cuts_and_batches_match_oracle(dtype):
    rig = rig_for(FULL, 6, device="cuda", dtype=dtype)
    t, u = toks(70, FULL["vocab"], 4), toks(40, FULL["vocab"], 8)
    want, wu = O.forward(FULL, rig.w, t), O.forward(FULL, rig.w, u)
    if dtype == torch.float32:
        cmp = lambda got, ref, which: close(got, ref)
    else:
        errs = {"t": _bf16_ref_err(FULL, rig.w, t, want), "u": _bf16_ref_err(FULL, rig.w, u, wu)}
        cmp = lambda got, ref, which: _bf16_close(got, ref, errs[which])
    for cuts in ([70], [2, 2, 3, 16, 1, 31], [33, 2, 2, 2], [20, 20], []):
        cmp(rig.run_cut("a", t, cuts), want, "t")
    a = rig.step([("a", t[:30]), ("b", u[:5])])
    b = rig.step([("a", t[30:31]), ("b", u[5:])], end=["b"])
    c = rig.step([("a", t[31:])], end=["a"])
    cmp(torch.cat([a["a"], b["a"], c["a"]]), want, "t")
    cmp(torch.cat([a["b"], b["b"]]), wu, "u")


@pytest.mark.gpu
def test_gpu_layers_and_mechanisms_fp32():
    rig = rig_for(FULL, 5, device="cuda", dtype=torch.float32)
    t = toks(19, FULL["vocab"], 3)
    rig.model.layer_probe = []
    rig.run_cut("a", t, [19])
    for got, want in zip(rig.model.layer_probe, O.layers_of(FULL, rig.w, t)):
        close(got.cpu(), want)
    rig.model.layer_probe = None
    for name, layers in SINGLE.items():
        cfg = make_cfg(layers)
        r2 = rig_for(cfg, 3, device="cuda", dtype=torch.float32)
        u = toks(45, cfg["vocab"], 1)
        close(r2.run_cut("a", u, [20, 2]), O.forward(cfg, r2.w, u))


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_gpu_odd_sizes(dtype):
    rig = rig_for(ODD, 31, device="cuda", dtype=dtype)
    t = toks(41, 53, 3)
    want = O.forward(ODD, rig.w, t)
    ref = _bf16_ref_err(ODD, rig.w, t, want) if dtype == torch.bfloat16 else None
    for cuts in ([41], [3, 2, 17]):
        got = rig.run_cut("a", t, cuts)
        close(got, want) if dtype == torch.float32 else _bf16_close(got, want, ref)


BIG = make_cfg([par(att(8, 2, 64, 64, 0.125, 20.0, 50, 64, 1e4), delta(4, 2, 32, 64, 4), mlp=dense(192)), mamba(256, 16, 4, 8, mlp=dense(160)),
                wkv(4, 32, 16, mlp=dense(96)), par(att(4, 2, 128, 128, 0.09, 30.0, 96, 32, 1e6), delta(2, 2, 128, 128, 4)), wkv(2, 64, 8),
                par(att(4, 4, 64, 128, 0.125, 25.0, 33, 32, 1e4), delta(4, 4, 64, 32, 4)),
                par(att(8, 1, 128, 64, 0.09, 15.0, 200, 128, 1e5), delta(2, 1, 48, 40, 2)), mamba(200, 40, 3, 16)], width=128, vocab=211, share=(1, 0))


@pytest.mark.gpu
def test_gpu_matrix_core_sizes_bf16():
    """Head sizes of 64 / 128 take the matrix-core attention kernels and the vector decode kernels; long
    enough for several chunks, pages per wave and tiles of the scans."""
    rig = rig_for(BIG, 6, device="cuda", dtype=torch.bfloat16, num_blocks=48)
    t = toks(150, BIG["vocab"], 4)
    want = O.forward(BIG, rig.w, t)
    ref = _bf16_ref_err(BIG, rig.w, t, want, num_blocks=48)
    for cuts in ([150], [2, 2, 3, 16, 1, 31], [100]):
        _bf16_close(rig.run_cut("a", t, cuts), want, ref)
    r32 = rig_for(BIG, 6, device="cuda", dtype=torch.float32, num_blocks=48)
    close(r32.run_cut("a", t, [70, 3]), want)


@pytest.mark.gpu
def test_gpu_long_prompt_fp32_and_bf16():
    """600 tokens (38 pages and tiles of the scans), whole and cut so that the second portion and the
    decoded tokens read the caches and the states."""
    cfg = make_cfg(BIG["layers"][:3], width=128, vocab=211)
    t = toks(600, cfg["vocab"], 4)
    w = O.random_weights(cfg, 7)
    want = O.forward(cfg, w, t)
    r32 = rig_for(cfg, w=w, device="cuda", dtype=torch.float32, num_blocks=96)
    close(r32.run_cut("a", t, [600]), want)
    close(r32.run_cut("a", t, [413, 180]), want)
    rig = rig_for(cfg, w=w, device="cuda", dtype=torch.bfloat16, num_blocks=96)
    _bf16_close(rig.run_cut("a", t, [500, 95]), want, _bf16_ref_err(cfg, w, t, want, num_blocks=96))


@pytest.mark.gpu
def test_gpu_far_tokens_and_chunk_edges():
    for kind in ("mamba", "wkv", "delta"):
        cfg, w, t, far, n = _slow_state(kind)
        want = O.forward(cfg, w, t)
        for cuts in ([n], [310], [100, 2, 64, 130]):
            close(rig_for(cfg, w=w, num_blocks=32, device="cuda").run_cut("a", t, cuts), want, tol=1e-4)
    for dims, dtype in ((8, torch.float32), (64, torch.float32), (64, torch.bfloat16)):
        for chunk in (1, 15, 16, 17, 48):
            cfg = make_cfg([par(att(2, 1, dims, dims, 0.2, chunk=chunk, dims=4))], width=24, vocab=37)
            far = 2 * chunk - 1
            n = far + chunk + 4
            w, t = _spiked(cfg, 11, far, n, ("l0.mix.left.v",))
            w = _only(cfg, "left")(w)
            want = O.forward(cfg, w, t)
            for cuts in ([n], [far], [far + 1], [2] * (n // 2 + 1)):
                got = rig_for(cfg, w=w, device="cuda", dtype=dtype).run_cut("a", t, cuts)
                if dtype == torch.float32:
                    close(got, want, tol=1e-4)
                else:  # a key seen one position too long or too short moves a row by far more than this
                    assert float(_row_err(got, want).max()) < 0.04
                    d = (want - _moved(cfg, w, t, far))[far].pow(2).mean().sqrt() / want.pow(2).mean().sqrt()
                    assert float(d) > 0.2


@pytest.mark.gpu
def test_gpu_unequal_batch_and_reuse_fp32():
    rig = rig_for(FULL, 9, num_blocks=12, device="cuda")
    T = _plan_tokens(FULL["vocab"])
    got = _run_plans(rig, T)
    for n in T:
        close(got[n], O.forward(FULL, rig.w, T[n]))


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_gpu_norm_and_mix_ops_match_their_torch_forms(dtype):
    g = torch.Generator().manual_seed(3)
    tol = 1e-5 if dtype == torch.float32 else 2e-2
    rnd = lambda *s: torch.randn(*s, generator=g)
    for T, d in ((5, 24), (3, 7), (2, 1), (4, 520), (3, 1028), (2, 2052), (2, 4100), (2, 8192), (3, 301), (2, 2051)):
        x, a, b = rnd(T, d) * 2 + 0.5, (rnd(T, d) * 3 + 1).to(dtype), rnd(T, d).to(dtype)
        p, q, ws = (rnd(d), rnd(d)), (rnd(d), rnd(d)), (rnd(d), rnd(d))
        for branch, pre, kw in (((), q, {}), ((a,), q, {}), ((a,), None, {}), ((a, b), q, dict(branch_w=ws, mix=0.5)), ((a.float(), b), q, dict(branch_w=ws, mix=2.0))):
            cu = lambda v: tuple(t.cuda() for t in v) if v is not None else None
            xc, xg = x.clone(), x.cuda()
            want = hops.join_norm(xc, branch, p, pre, 1e-5, dtype, **kw)
            got = hops.join_norm(xg, cu(branch), cu(p), cu(pre), 1e-5, dtype, **{k: cu(v) if k == "branch_w" else v for k, v in kw.items()})
            close(xg.cpu(), xc.double(), tol=2e-5)
            assert (got is None) == (want is None)
            if want is not None:
                close(got.cpu().float(), want.double(), tol=tol)
    for d, n in ((24, 5), (7, 5), (1030, 2), (1028, 8), (1, 1)):
        cu_, ctx, slot = _i32(0, 1, 4, 5, 9, 10), _i32(3, 0, 0, 7, 2), _i32(2, 0, 1, -1, 4)
        h, mu, st = rnd(10, d), rnd(n, d), rnd(5, d)
        sg = st.cuda()
        want = hops.token_mix(h, mu, st, cu_, ctx, slot, dtype)
        got = hops.token_mix(h.cuda(), mu.cuda(), sg, cu_.cuda(), ctx.cuda(), slot.cuda(), dtype)
        live = [0, 1, 2, 3, 4, 9]  # rows of padding segments are nobody's
        close(got.cpu().float()[live], want.double()[live], tol=tol)
        assert torch.equal(sg.cpu(), st)
    for kind in ("relu_sq", "tanh"):
        z = (rnd(5, 27) * 2).to(dtype)
        close(hops.activation(z.cuda(), kind).cpu().float(), hops.activation(z, kind).double(), tol=tol)


LENS = [1, 15, 16, 17, 100, 7, 33, 32, 31]


def _segments():
    cu = torch.tensor([0] + list(torch.tensor(LENS).cumsum(0)), dtype=torch.int32)
    return cu, _i32(0, 5, 0, 64, 0, 3, 9, 0, 2), _i32(0, 1, 2, 3, 4, -1, 5, 7, 6)


def _both_devices(fn, state, inputs):
    """fn(state, seg, *inputs) on CPU copies and on the GPU; outputs and states must agree."""
    seg = _segments()
    sc, sg = state.clone(), state.cuda()
    want = fn(sc, seg, *inputs)
    got = fn(sg, tuple(s.cuda() for s in seg), *[i.cuda() if isinstance(i, torch.Tensor) else i for i in inputs])
    close(got.cpu().float(), want.double(), tol=2e-5)
    close(sg.cpu(), sc.double(), tol=2e-5)
    return got.cpu()


@pytest.mark.gpu
@pytest.mark.parametrize("C,N", [(64, 16), (70, 8), (33, 5), (1, 1), (130, 24), (48, 32), (40, 33), (24, 64), (20, 100), (12, 200), (9, 256), (200, 12)])
def test_gpu_selective_scan_matches_the_recurrence(C, N):
    """Segments shorter than, equal to and longer than the kernel's tiles, some continuing from their
    slots, one padding segment, slots with leftovers; outputs and states."""
    g = torch.Generator().manual_seed(5)
    (xc, q, dt, db, al, D, pr), want = _scan_case(g, sum(LENS), C, N)
    st = torch.randn(8, C, N, generator=g) * 0.3
    got = _both_devices(lambda s, seg, *a: hops.selective_scan(a[0], a[1], 3, 3 + N, *a[2:], C, s, *seg), st, (xc, q, dt, db, al, D, pr))
    a, b = sum(LENS[:4]), sum(LENS[:5])  # the 100-token segment starts from zero: the written-out recurrence
    y = O.selective_scan(xc[a:b].double(), O.softplus(dt[a:b].double() + db.double()), -torch.exp(al.double()), q[a:b, 3:3 + N].double(),
                         q[a:b, 3 + N:].double(), D.double()) * O.silu(pr[a:b, C:].double())
    close(got[a:b], y, tol=2e-5)


@pytest.mark.gpu
@pytest.mark.parametrize("mean", [-14.0, -5.0, 3.0, 25.0])
def test_gpu_selective_scan_step_sizes(mean):
    """Step sizes from millionths to tens: the kernel's softplus in each of its ranges."""
    g = torch.Generator().manual_seed(6)
    (xc, q, dt, db, al, D, pr), want = _scan_case(g, 40, 20, 4, mean)
    D = torch.zeros(20)
    y = O.selective_scan(xc.double(), O.softplus(dt.double() + db.double()), -torch.exp(al.double()), q[:, 3:7].double(), q[:, 7:].double(),
                         D.double()) * O.silu(pr[:, 20:].double())
    st = torch.zeros(1, 20, 4, device="cuda")
    got = hops.selective_scan(*[v.cuda() for v in (xc, q)], 3, 7, *[v.cuda() for v in (dt, db, al, D, pr)], 20, st, *[_i32(*v).cuda() for v in ((0, 40), (0,), (0,))])
    assert float((got.cpu().double() - y).abs().max() / y.abs().max()) < 3e-6


@pytest.mark.gpu
@pytest.mark.parametrize("H,Gk,dk,dv", [(2, 2, 32, 32), (4, 2, 48, 32), (3, 1, 64, 96), (2, 2, 128, 128), (1, 1, 200, 40), (6, 3, 5, 7),
                                        (2, 1, 16, 8), (1, 1, 1, 1), (2, 2, 256, 16), (3, 3, 36, 130), (2, 2, 100, 9)])
def test_gpu_delta_rule_and_bonus_match_the_recurrence(H, Gk, dk, dv):
    """One decay per head with the delta rule, and the current-token bonus: both forms of the scan."""
    g = torch.Generator().manual_seed(7)
    T, a, b = sum(LENS), sum(LENS[:4]), sum(LENS[:5])
    qkv, zb, kw, _ = _delta_case(g, T, H, Gk, dk, dv)
    alone = _delta_alone(qkv[a:b], zb, kw, H, Gk, dk, dv)
    st = torch.randn(8, H, dv, dk, generator=g) * 0.3
    a_log = kw.pop("a_log")
    for mode in (1, 2):
        got = _both_devices(lambda s, seg, x, z, al: hops.decay_scan(x, 0, Gk * dk, 2 * Gk * dk, x, z, s, *seg, H, Gk, dk, dv, dk ** -0.5, a_log=al,
                                                                     beta=x, mode=mode, **kw), st, (qkv, zb, a_log))
        close(got[a:b], alone, tol=2e-5)
    rkv, z, w0, u, _ = _wkv_case(g, T, H, dk)
    n = H * dk
    r, k, v = (rkv[a:b, i * n:(i + 1) * n].double().view(b - a, H, dk) for i in range(3))
    alone = O.wkv_scan(r, k, v, torch.exp(-torch.exp(z[a:b].double() + w0.double())).view(b - a, H, dk), u.double()).reshape(b - a, n)
    st = torch.randn(8, H, dk, dk, generator=g) * 0.3
    for mode in (1, 2):
        got = _both_devices(lambda s, seg, *x: hops.decay_scan(x[0], 0, n, 2 * n, x[1], x[2], s, *seg, H, H, dk, dk, 1.0, decay="exp_exp", bonus=x[3],
                                                               mode=mode), st, (rkv, z, w0, u))
        close(got[a:b], alone, tol=2e-5)


def _delta_alone(qkv, zb, kw, H, Gk, dk, dv):
    """The delta rule written out for given rows [q | k | v | beta | a], as one sequence."""
    n, c = qkv.shape[0], kw["beta_col"]
    x = qkv.double()
    unit = lambda v: v / torch.sqrt((v * v).sum(-1, keepdim=True) + 1e-6)
    q, k = unit(x[:, :Gk * dk].view(n, Gk, dk)) * dk ** -0.5, unit(x[:, Gk * dk:2 * Gk * dk].view(n, Gk, dk))
    v, beta = x[:, 2 * Gk * dk:c].view(n, H, dv), torch.sigmoid(x[:, c:c + H])
    dec = torch.exp(-torch.exp(kw["a_log"].double()) * O.softplus(x[:, c + H:] + zb.double()))
    out = torch.zeros(n, H, dv, dtype=torch.float64)
    for h in range(H):
        S, j = torch.zeros(dk, dv, dtype=torch.float64), h // (H // Gk)
        for t in range(n):
            S = dec[t, h] * S
            S = S + torch.outer(k[t, j], beta[t, h] * (v[t, h] - S.T @ k[t, j]))
            out[t, h] = S.T @ q[t, j]
    return out.reshape(n, H * dv)


@pytest.mark.gpu
@pytest.mark.parametrize("Hq,G,dk,dv", [(4, 2, 64, 64), (2, 1, 128, 128), (8, 1, 64, 128), (2, 2, 128, 64), (6, 2, 24, 40), (3, 3, 7, 5)])
def test_gpu_chunked_capped_attention_kernels(Hq, G, dk, dv):
    """Prompt portions and decode rows, matrix-core / vector / any-size kernels, chunks below, at and above
    the page size, scores near the cap."""
    g = torch.Generator().manual_seed(8)
    n = 90
    qkv = (torch.randn(n, Hq * dk + G * dk + G * dv, generator=g) * 2).to(torch.bfloat16).float()
    q, k = qkv[:, :Hq * dk].double().view(n, Hq, dk), qkv[:, Hq * dk:Hq * dk + G * dk].double().view(n, G, dk)
    v = qkv[:, Hq * dk + G * dk:].double().view(n, G, dv)
    kc, vc = torch.zeros(8, 16, G * dk), torch.zeros(8, G, dv, 16)
    order = [2, 0, 7, 3, 5, 1]
    for t in range(n):
        kc[order[t // 16], t % 16] = k[t].float().reshape(-1)
        vc[order[t // 16], :, :, t % 16] = v[t].float()
    bt = _i32(*order).view(1, 6).cuda()
    scale = 2.0 * dk ** -0.5 / 4
    for dtype, tol in ((torch.float32, 2e-5), (torch.bfloat16, 2e-2)):
        x, kd, vd = qkv.cuda().to(dtype), kc.cuda().to(dtype), vc.cuda().to(dtype)
        for size, cap in ((1, 5.0), (13, 2.0), (16, 1.0), (17, 3.0), (64, 0.5), (90, 30.0), (500, 4.0), (40, 90.0)):
            want = O.chunked_attention(q, k, v, scale, cap, size)
            kw = dict(chunked=True, cap=cap)
            for a, b in ((0, 90), (5, 7), (15, 64)):
                for fast in ((0, 1) if dtype == torch.bfloat16 and dk < 64 else (0, 16, 32, 64)):
                    got = hops.window_attention_prefill(x[a:b].contiguous(), kd, vd, _i32(0, b - a).cuda(), _i32(a).cuda(), bt, Hq, G, dk, dv, scale,
                                                        size, False, mfma=fast, **kw)
                    close(got.cpu().float(), want[a:b], tol=tol)
            for t in (0, 12, 13, 16, 63, 64, 89):
                for vec in (True, False):
                    got = hops.window_attention_decode(x[t:t + 1], kd, vd, bt, _i32(t + 1).cuda(), Hq, G, dk, dv, scale, size, False, vec=vec, **kw)
                    close(got.cpu().float(), want[t:t + 1], tol=tol)


@pytest.mark.gpu
def test_gpu_greedy_generation_with_graphs():
    eng = LLMEngine(EngineConfig(model="dopivik-tiny", max_num_seqs=4, max_model_len=256, num_blocks=64,
                                 dtype="float32", max_prefill_tokens=32, mixed_prefill_tokens=16), device="cuda")
    eng.warmup()  # decode steps replay from captured hipGraphs
    cfg, w = hybrid_config_to_dict(eng.model_cfg), {k: v.cpu() for k, v in state_dict(eng.model).items()}
    prompts = [toks(n, 336, 40 + n) for n in (5, 37, 21)]
    seqs = eng.generate(prompts, SamplingParams(max_tokens=12, temperature=0.0, ignore_eos=True))
    assert eng.stats()["graph_buckets"]
    for p, s in zip(prompts, seqs):
        assert s.output_ids == O.greedy(cfg, w, p, 12)
