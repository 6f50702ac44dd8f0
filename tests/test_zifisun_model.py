"""The Zifisun layer-list design in the engine against the plain float64 oracle
(tests/zifisun_oracle.py): each mechanism alone (several residual streams, windowed attention that keeps
the first tokens visible, latent attention, per-head gates, the corrected group-limited router with
identity experts), prefill against token-by-token decoding, prompt portions down to two tokens, unequal
batches, pages that are reused, keys just inside and outside a window, among the kept first ones and
right behind them, at page borders and hundreds of tokens away, the first tokens, looped layers with a
cache per pass, long decoding, odd sizes and sizes of one, and greedy generation through the engine and
the trace command.

Runs on the CPU (the ops' torch forms); the ``gpu`` tests at the end run the same comparisons
through the HIP kernels."""
import copy
import json
import subprocess
import sys

import numpy as np
import pytest
import torch

import zifisun_oracle as O
from k8s_llm_monitor_amd.engine import EngineConfig, LLMEngine, SamplingParams
from k8s_llm_monitor_amd.models.config import get_config, hybrid_config_from_dict, hybrid_config_to_dict
from k8s_llm_monitor_amd.models.hybrid import state_dict
from k8s_llm_monitor_amd.models.registry import build_model, config_from_dir
from k8s_llm_monitor_amd.ops import hybrid as hops
from test_hybrid_model import ROOT, Rig, _save, close, toks
from test_levovik_model import _bf16_close, _row_err


# ------------------------------------------------------------------ small configurations

def att(heads=4, kv=2, dim=10, vdim=6, scale=0.35, size=12, keep=3, mlp=None):
    return {"type": "attention", "mixer": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale,
                                           "mask": {"size": size, "keep_first": keep}}, "mlp": mlp}


def lat(heads=3, dim=8, rot=6, vdim=10, q_rank=14, kv_rank=12, scale=0.3, size=17, base=100.0, mlp=None):
    return {"type": "latent_attention", "mixer": {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "q_rank": q_rank,
                                                  "kv_rank": kv_rank, "scale": scale, "mask": {"size": size},
                                                  "rot": {"base": base, "dims": rot}}, "mlp": mlp}


def moe(experts=6, top=2, ff=14, shared=20, identity=2, groups=(2, 1)):
    r = {"experts": experts, "top": top}
    if identity is not None:
        r["identity"] = identity
    if groups is not None:
        r["groups"] = {"count": groups[0], "keep": groups[1]}
    return {"kind": "moe", "expert": {"ff": ff}, "router": r, "shared": {"ff": shared} if shared else None}


def make_cfg(layers, width=36, vocab=59, streams=3, eps=1e-6, loop=None):
    c = {"architecture": "Zifisun", "vocab": vocab, "width": width, "layers": layers, "norm": {"eps": eps}, "streams": streams}
    if loop:
        c["loop"] = dict(zip(("start", "stop", "times"), loop))
    return c


FULL = make_cfg([att(mlp=moe()), lat(mlp=moe(5, 3, 9, 0, 3, (2, 1))), att(2, 1, 16, 12, 0.25, 20, 18), lat(4, 6, 4, 5, 11, 9, 0.4, 9, 1e4, mlp=moe(4, 1, 8, 12, None, None))],
                loop=(1, 3, 2))


def rig_for(cfg, seed=0, w=None, **kw):
    return Rig(dict(cfg, max_positions=kw.pop("max_positions", 1024)), w=w if w is not None else O.random_weights(cfg, seed), **kw)


# ------------------------------------------------------------------ mechanisms alone

SINGLE = {
    "attention": [att()], "attention-no-kept": [att(keep=0)], "attention-kept-beyond-prompt": [att(keep=100)],
    "attention-window-1": [att(size=1, keep=1)], "attention-window-beyond-prompt": [att(size=500, keep=4)],
    "attention-kept-over-pages": [att(size=7, keep=21)], "attention-ones": [att(1, 1, 1, 1, 1.0, 1, 1)],
    "attention-mqa": [att(5, 1, 6, 9)], "attention-own-keys": [att(3, 3, 7, 4, size=16, keep=16)],
    "latent": [lat()], "latent-ones": [lat(1, 1, 2, 1, 1, 1, 1.0, 1)], "latent-window-1": [lat(size=1)],
    "latent-window-beyond-prompt": [lat(size=400)], "latent-wide-heads": [lat(7, 5, 10, 3, 4, 20, size=16)],
    "moe": [att(mlp=moe())], "moe-one-group": [att(mlp=moe(groups=None))], "moe-no-identity": [att(mlp=moe(identity=None, groups=(3, 1)))],
    "moe-mostly-identity": [lat(mlp=moe(2, 2, 7, 9, 10, (3, 2)))], "moe-no-shared": [lat(mlp=moe(shared=0))],
    "moe-one-of-one": [lat(mlp=moe(1, 1, 1, 1, 0, (1, 1)))], "moe-groups-of-one": [att(mlp=moe(4, 3, 8, 5, 2, (6, 3)))],
    "moe-all": [lat(mlp=moe(3, 4, 6, 10, 1, (2, 2)))]}


@pytest.mark.parametrize("name", list(SINGLE))
def test_single_mechanism_whole_prompt(name):
    cfg = make_cfg(SINGLE[name])
    rig = rig_for(cfg, 3)
    t = toks(40, cfg["vocab"], 1)
    close(rig.run_cut("a", t, [40]), O.forward(cfg, rig.w, t))


@pytest.mark.parametrize("streams", [1, 2, 4, 7])
def test_streams(streams):
    cfg = make_cfg([att(mlp=moe()), lat()], streams=streams)
    rig = rig_for(cfg, 4)
    t = toks(24, cfg["vocab"], 2)
    want = O.forward(cfg, rig.w, t)
    for cuts in ([24], [5, 2]):
        close(rig.run_cut("a", t, cuts), want)


ODD = make_cfg([att(5, 5, 7, 3, 0.5, 11, 5, mlp=moe(3, 2, 11, 7, 2, (5, 3))), lat(3, 5, 2, 7, 9, 13, 0.5, 7, mlp=moe(5, 2, 3, 0, 1, (3, 2))),
                att(6, 2, 11, 13, 0.3, 16, 17)], width=37, vocab=53, streams=5, loop=(0, 2, 3))


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
    assert len(rig.model.layer_probe) == layers.shape[0] == 6
    for got, want in zip(rig.model.layer_probe, layers):
        close(got, want)
    rig.model.layer_probe = None


def test_stream_op_against_the_written_out_sums():
    g = torch.Generator().manual_seed(1)
    rnd = lambda *s: torch.randn(*s, generator=g)
    for S in (1, 3, 4):
        x, y, mix, out, read, w = rnd(5, S, 12), rnd(5, 12), rnd(S, S), rnd(S), rnd(S), rnd(12)
        xs = x.double().transpose(0, 1)
        new = O.write_streams(xs, mix.double(), out.double(), y.double())
        buf = x.clone()
        h, xn = hops.stream_norm(buf, y, (mix, out), read, w, 1e-6, torch.float32, S)
        assert xn is buf
        close(buf, new.transpose(0, 1), tol=1e-6)
        close(h, O.rms_norm(O.read_streams(new, read.double()), w.double(), 1e-6), tol=1e-6)
        buf = x.clone()
        h, xn = hops.stream_norm(buf, None, None, None, w, 1e-6, torch.float32, S)
        assert xn is buf and torch.equal(buf, x)
        close(h, O.rms_norm(xs.sum(0), w.double(), 1e-6), tol=1e-6)
        one = x[:, :1].contiguous()  # one row that stands for all streams
        keep = one.clone()
        h, xn = hops.stream_norm(one, y, (mix, out), read, w, 1e-6, torch.float32, S)
        new = O.write_streams(keep.double().transpose(0, 1).expand(S, 5, 12), mix.double(), out.double(), y.double())
        assert S == 1 or torch.equal(one, keep)
        close(xn, new.transpose(0, 1), tol=1e-6)
        close(h, O.rms_norm(O.read_streams(new, read.double()), w.double(), 1e-6), tol=1e-6)


# (experts, top, groups, keep) of the router cases
ROUTES = [(8, 2, 2, 1), (12, 2, 2, 1), (12, 3, 4, 2), (6, 6, 1, 1), (9, 2, 9, 4), (16, 5, 4, 3), (40, 4, 8, 2), (70, 8, 7, 3), (256, 16, 16, 5), (1, 1, 1, 1)]


def _route_case(E, d, n, seed, shift):
    g = torch.Generator().manual_seed(seed)
    return torch.randn(n, d, generator=g), torch.randn(E, d, generator=g) * d ** -0.5 * 2, torch.randn(E, generator=g) * 0.3 + shift


def _route_want(h, wr, corr, K, groups, keep):
    ids, wts = [], []
    for t in range(h.shape[0]):
        s = O.softmax(wr.double() @ h[t].double())
        e = O.route(s, corr.double(), K, groups, keep)
        ids.append(e)
        wts.append(s[e])
    return torch.tensor(ids, dtype=torch.int32), torch.stack(wts)


@pytest.mark.parametrize("E,K,groups,keep", ROUTES)
@pytest.mark.parametrize("shift", [0.0, -2.0])
def test_router_choice(E, K, groups, keep, shift):
    """Corrections move the choice (with ``shift`` all choice scores are negative: experts outside the kept
    groups must not win with a zero), the weights stay the softmax scores."""
    h, wr, corr = _route_case(E, 20, 9, E, shift)
    ids, wts = hops.moe_router_grouped(h, wr, E, K, groups, keep, 1.0, soft=True, corr=corr, best2=False, renorm=False)
    wi, ww = _route_want(h, wr, corr, K, groups, keep)
    assert torch.equal(ids, wi)
    close(wts, ww, tol=1e-5)


def _keep_case(g, n, H, G, dk, dv):
    """Rows [q | k | v | H gate logits | 3 more], pages of one sequence and the gated outputs' inputs."""
    qkv = torch.randn(n, H * dk + G * dk + G * dv + H + 3, generator=g) * 1.3
    q, k = qkv[:, :H * dk].double().view(n, H, dk), qkv[:, H * dk:H * dk + G * dk].double().view(n, G, dk)
    v = qkv[:, H * dk + G * dk:H * dk + G * dk + G * dv].double().view(n, G, dv)
    kc, vc = torch.zeros(8, 16, G * dk), torch.zeros(8, G, dv, 16)
    order = [2, 0, 7, 3, 5, 1]
    for t in range(n):
        kc[order[t // 16], t % 16] = k[t].float().reshape(-1)
        vc[order[t // 16], :, :, t % 16] = v[t].float()
    col = H * dk + G * dk + G * dv
    return qkv, q, k, v, kc, vc, torch.tensor([order], dtype=torch.int32), col


def _keep_want(q, k, v, qkv, col, scale, size, keep):
    n, H = q.shape[:2]
    o = O.attend(q, k, v, scale, size, keep)
    return (o * torch.sigmoid(qkv[:, col:col + H].double()).unsqueeze(-1)).reshape(n, -1)


def _i32(*a):
    return torch.tensor(a, dtype=torch.int32)


MASKS = ((1, 0), (1, 1), (7, 3), (16, 16), (17, 15), (20, 40), (64, 5), (5, 33), (500, 4), (3, 90))


def test_kept_first_tokens_and_gate_op():
    """Prompt portions and single decode rows over the pages against the written-out attention."""
    g = torch.Generator().manual_seed(4)
    H, G, dk, dv, n = 4, 2, 6, 5, 84
    qkv, q, k, v, kc, vc, bt, col = _keep_case(g, n, H, G, dk, dv)
    for size, keep in MASKS:
        want = _keep_want(q, k, v, qkv, col, 0.4, size, keep)
        kw = dict(keep=keep, g_col=col)
        for a, b in ((0, n), (5, 7), (15, 34)):
            x = qkv[a:b].contiguous()
            got = hops.window_attention_prefill(x, kc, vc, _i32(0, b - a), _i32(a), bt, H, G, dk, dv, 0.4, size, False, gate=x, **kw)
            close(got, want[a:b], tol=1e-5)
        for t in (0, 6, 15, 16, 33, 83):
            x = qkv[t:t + 1]
            got = hops.window_attention_decode(x, kc, vc, bt, _i32(t + 1), H, G, dk, dv, 0.4, size, False, gate=x, **kw)
            close(got, want[t:t + 1], tol=1e-5)


# ------------------------------------------------------------------ cuts, decoding, batches

def test_prefill_equals_token_by_token_and_portions():
    rig = rig_for(FULL, 6)
    t = toks(70, FULL["vocab"], 4)
    want = O.forward(FULL, rig.w, t)
    for cuts in ([70], [], [2, 2, 3, 16, 1, 31], [15, 17, 16, 2], [33, 2, 2, 2], [20, 20, 20]):
        close(rig.run_cut("a", t, cuts), want)


def test_first_tokens_and_single_token_prompt():
    rig = rig_for(FULL, 7)
    for n in (1, 2, 3, 4):
        t = toks(n, FULL["vocab"], 10 + n)
        close(rig.run_cut("a", t, [n]), O.forward(FULL, rig.w, t))
        close(rig.run_cut("a", t, []), O.forward(FULL, rig.w, t))


def test_long_decoding_over_pages_and_windows():
    rig = rig_for(FULL, 8)
    t = toks(130, FULL["vocab"], 5)
    close(rig.run_cut("a", t, [10]), O.forward(FULL, rig.w, t))  # 120 decode steps over 8 pages


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
    """Live requests with portions beside decode tokens; one ends and its pages are taken by a new request
    whose logits must not see what they held."""
    rig = rig_for(FULL, 9, num_blocks=12)
    T = _plan_tokens(FULL["vocab"])
    got = _run_plans(rig, T)
    for n in T:
        close(got[n], O.forward(FULL, rig.w, T[n]))
    assert rig.blocks.num_free == 12


def test_every_pass_of_a_loop_has_its_own_cache():
    base = [att(size=6, keep=2, mlp=moe()), lat(size=9)]
    looped = make_cfg(base, loop=(0, 2, 3))
    w = O.random_weights(looped, 4)
    plain = make_cfg(base * 3)
    wp = dict(w)
    for i in range(2, 6):
        wp.update({f"l{i}." + k[len(f"l{i % 2}."):]: v for k, v in w.items() if k.startswith(f"l{i % 2}.")})
    t = toks(40, looped["vocab"], 2)
    want = O.forward(looped, w, t)
    close(O.forward(plain, wp, t), want, tol=1e-12)
    a, b = rig_for(looped, w=w), rig_for(plain, w=wp)
    for cuts in ([40], [7, 2, 20]):
        close(a.run_cut("a", t, cuts), want)
        close(b.run_cut("a", t, cuts), want)
    assert len(a.runner.kv) == 6 and a.model.cache_bytes() == b.model.cache_bytes()
    assert a.model.resident_weight_bytes() < b.model.resident_weight_bytes()


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


@pytest.mark.parametrize("size", [1, 2, 15, 16, 17, 24])
@pytest.mark.parametrize("kind", ["attention", "latent"])
def test_window_edges(kind, size):
    """A spiked key is seen by exactly the ``size`` positions from its own on, wherever the prompt is cut and
    whether those positions are prefilled or decoded."""
    layer, name = (att(2, 1, 8, 8, size=size, keep=2), "v") if kind == "attention" else (lat(2, 8, 4, 8, 12, 10, size=size), "uv")
    cfg = make_cfg([layer], width=24, vocab=37)
    for far in (4, 15, 16):
        n = far + size + 4
        w, t = _spiked(cfg, 11, far, n, ("l0.mix." + name,))
        want, other = O.forward(cfg, w, t), _moved(cfg, w, t, far)
        end = far + size  # the first position that must not see it
        d = (want - other).abs().amax(-1)
        assert all(float(d[p]) > 1e-3 for p in range(far, end)) and all(float(d[p]) < 1e-12 for p in range(end, n))
        for cuts in ([n], [far], [far + 1], [end], [max(1, end - 1), 2], [2] * (n // 2 + 1)):
            close(rig_for(cfg, w=w).run_cut("a", t, cuts), want, tol=1e-4)


@pytest.mark.parametrize("keep", [1, 3, 15, 16, 17, 33])
def test_kept_first_edges(keep):
    """The last kept position is seen by every later one, the next position only within the window."""
    cfg = make_cfg([att(2, 1, 8, 8, size=6, keep=keep)], width=24, vocab=37)
    n = keep + 30
    for far in (0, keep - 1, keep):
        w, t = _spiked(cfg, 12, far, n, ("l0.mix.v",))
        want, other = O.forward(cfg, w, t), _moved(cfg, w, t, far)
        d = (want - other).abs().amax(-1)
        seen = [p >= far and (far < keep or p - far < 6) for p in range(n)]
        assert all((float(d[p]) > 1e-3) == s and (s or float(d[p]) < 1e-12) for p, s in enumerate(seen))
        for cuts in ([n], [keep], [keep + 1, 2], [keep + 8], [2] * (n // 2 + 1), [1]):
            close(rig_for(cfg, w=w).run_cut("a", t, cuts), want, tol=1e-4)


def _marked(cfg, seed, far, n):
    """Axis 0 of the embedding is the same for all tokens, axis 1 marks the special one."""
    w, t = _spiked(cfg, seed, far, n)
    e = w["embed"]
    e[:, 0], e[:, 1] = 1.0, 0.0
    e[cfg["vocab"] - 1, 1] = 4.0
    w["l0.norm1"] = torch.ones(cfg["width"])
    return w, t, torch.eye(cfg["width"])


def _peaked(kind, far, n, size, keep=0, dims=8):
    """A one-layer model in which the special key takes most of every later query's softmax."""
    layer = att(2, 1, dims, dims, 0.5, size, keep) if kind == "attention" else lat(2, dims, 4, dims, 12, 10, 1.0, size, 1e4)
    cfg = make_cfg([layer], width=24, vocab=37)
    w, t, eye = _marked(cfg, 13, far, n)
    if kind == "attention":
        for h in range(2):
            w["l0.mix.q"][h * dims + dims - 1] = 8.0 * eye[0]
        w["l0.mix.k"][dims - 1] = 8.0 * eye[1]
        w["l0.mix.q.norm"], w["l0.mix.k.norm"] = torch.full((dims,), 2.0), torch.full((dims,), 1.5)
    else:
        w["l0.mix.dq"][0], w["l0.mix.dkv"][0] = 8.0 * eye[0], 8.0 * eye[1]
        for h in range(2):
            w["l0.mix.uq"][h * (dims + 4), 0], w["l0.mix.uk"][h * dims, 0] = 3.0, 1.0
    return cfg, w, t


@pytest.mark.parametrize("kind", ["attention", "attention-kept", "latent"])
def test_far_key_with_a_peaked_score(kind):
    """One key takes a large part of the softmax of every later query that sees it, hundreds of tokens on."""
    n = 330
    if kind == "attention-kept":
        far, end = 2, n  # kept: seen to the end, far outside the window
        cfg, w, t = _peaked("attention", far, n, 40, 3)
    else:
        far, end = 20, 320
        cfg, w, t = _peaked(kind, far, n, 300)
    want = O.forward(cfg, w, t)
    d = (want - _moved(cfg, w, t, far)).abs().amax(-1)
    assert float(d[end - 1]) > 0.1 and all(float(x) < 1e-12 for x in d[end:])
    for cuts in ([n], [310], [100, 2, 64, 130], [far + 12]):
        close(rig_for(cfg, w=w, num_blocks=32).run_cut("a", t, cuts), want, tol=1e-4)


def test_every_tensor_and_constant_matters_and_is_read():
    """The oracle moves when any tensor or constant is changed, and the engine follows it."""
    cfg = make_cfg([att(4, 2, 8, 6, size=5, keep=2, mlp=moe(6, 2, 12, 10, 2, (2, 1))), lat(2, 6, 4, 5, 9, 7, size=6, mlp=moe(4, 2, 8, 6, 2, (2, 1)))],
                   width=24, vocab=37, loop=(0, 1, 2))
    w = O.random_weights(cfg, 16)
    t = toks(14, 37, 6)
    want = O.forward(cfg, w, t)
    g = torch.Generator().manual_seed(3)
    for name, v in w.items():
        w0 = dict(w)
        w0[name] = v + (4.0 if "correction" in name else 0.5) * v.abs().mean() * torch.randn(v.shape, generator=g)
        got = O.forward(cfg, w0, t)
        if ".mlp.e" not in name:  # a token may not reach every expert
            assert float((got - want).abs().max()) > 1e-4, name
        if "correction" in name or ".hc" in name:
            close(rig_for(cfg, w=w0).run_cut("a", t, [14]), got, tol=1e-4)
    variants = []
    for path, val in ((("layers", 0, "mixer", "scale"), 1.0), (("layers", 1, "mixer", "scale"), 1.0), (("layers", 0, "mixer", "mask", "size"), 6),
                      (("layers", 0, "mixer", "mask", "keep_first"), 3), (("layers", 1, "mixer", "mask", "size"), 5),
                      (("layers", 1, "mixer", "rot", "base"), 5.0), (("norm", "eps"), 0.1), (("layers", 0, "mlp", "router", "top"), 3),
                      (("layers", 0, "mlp", "router", "groups", "keep"), 2), (("layers", 1, "mlp", "router", "groups"), None),
                      (("layers", 0, "mlp", "router", "groups", "count"), 4), (("layers", 1, "mlp", "shared"), None),
                      (("loop",), None), (("loop", "times"), 3), (("loop", "stop"), 2)):
        c2 = copy.deepcopy(cfg)
        node = c2
        for k in path[:-1]:
            node = node[k]
        node[path[-1]] = val
        w2 = {k: v for k, v in w.items() if val is not None or path[-1] != "shared" or not k.startswith("l1.mlp.shared")}
        assert float((O.forward(c2, w2, t) - want).abs().max()) > 1e-3, path
        variants.append((c2, w2))
    for c, wc in [(cfg, w)] + variants:
        ref = O.forward(c, wc, t)
        for cuts in ([14], [3, 2]):
            close(rig_for(c, w=wc).run_cut("a", t, cuts), ref, tol=1e-4)


def test_positions_and_kept_tokens_count_from_zero_on_any_pages():
    """Positions count from 0 in every sequence whatever pages it gets; large positions keep their accuracy."""
    cfg = make_cfg([lat(2, 6, 8, 6, 12, 10, 0.5, 150, 20.0), att(2, 1, 8, 6, 0.5, 64, 5)], width=24, vocab=37)
    rig = rig_for(cfg, 15, num_blocks=48)
    t = toks(320, 37, 9)
    want = O.forward(cfg, rig.w, t)
    rig.step([("z", toks(90, 37, 1))])  # holds the first pages
    close(rig.run_cut("a", t, [150, 3, 140]), want, tol=5e-4)


# ------------------------------------------------------------------ engine entry points

def test_greedy_generation_through_engine(tmp_path):
    w = O.random_weights(FULL, 21)
    d = _save(tmp_path, FULL, w)
    assert config_from_dir(d).arch == "zifisun"
    eng = LLMEngine(EngineConfig(model=str(d), weights=str(d), max_num_seqs=3, max_model_len=256, num_blocks=40,
                                 dtype="float32", max_prefill_tokens=16, mixed_prefill_tokens=8), device="cpu")
    prompts = [toks(n, FULL["vocab"], 30 + n) for n in (4, 29, 18, 40)]  # 4 requests over 3 rows: one waits
    seqs = eng.generate(prompts, SamplingParams(max_tokens=10, temperature=0.0, ignore_eos=True))
    for p, s in zip(prompts, seqs):
        assert s.output_ids == O.greedy(FULL, w, p, 10)
    assert eng.stats()["mixed_steps"] > 0


def test_prefix_pages_are_reused_across_requests():
    """No recurrent state: a second request with the same first pages takes them from the prefix cache."""
    eng = LLMEngine(EngineConfig(model="zifisun-tiny", max_num_seqs=2, max_model_len=128, num_blocks=24, dtype="float32"), device="cpu")
    cfg, w = hybrid_config_to_dict(eng.model_cfg), state_dict(eng.model)
    shared = toks(35, 368, 3)
    par = SamplingParams(max_tokens=4, temperature=0.0, ignore_eos=True)
    for tail in (1, 2):
        p = shared + toks(5, 368, tail)
        assert eng.generate([p], par)[0].output_ids == O.greedy(cfg, w, p, 4)
    assert eng.runner.n_steps["prefill_context_tokens"] >= 32


def test_preset_round_trip_and_registry():
    c = get_config("zifisun-tiny")
    assert hybrid_config_from_dict(hybrid_config_to_dict(c), c.name) == c
    m = build_model(c, device="cpu", dtype=torch.float32)
    w = state_dict(m)
    assert w["l0.hc1.mix"].shape == (3, 3) and w["l1.mix.g"].shape == (3, 88) and w["l0.mix.g"].shape == (4, 88)
    assert w["l0.mlp.router"].shape == (8, 88) and w["l0.mlp.correction"].shape == (8,) and "l0.mlp.e6.up" not in w
    assert "l2.norm2" not in w and "l2.hc2.in" not in w and "loop.step" not in w and not m.has_state
    cfg = hybrid_config_to_dict(c)
    assert sorted(w) == sorted(O.random_weights(cfg)) and all(w[k].shape == v.shape for k, v in O.random_weights(cfg).items())
    eng = LLMEngine(EngineConfig(model="zifisun-tiny", max_num_seqs=2, max_model_len=128, num_blocks=16,
                                 dtype="float32"), device="cpu")
    p = toks(11, c.vocab_size, 1)
    s = eng.generate([p], SamplingParams(max_tokens=6, temperature=0.0, ignore_eos=True))[0]
    assert s.output_ids == O.greedy(cfg, w, p, 6)


def test_config_errors_are_loud():
    ok = O.random_weights(make_cfg([att(mlp=moe())]), 1)
    for bad in (att(4, 3), att(keep=-1), lat(rot=5), att(mlp=moe(groups=(3, 1))), att(mlp=moe(groups=(4, 5))), att(mlp=moe(6, 3, groups=(4, 1))),
                att(mlp=moe(top=9)), att(mlp={"kind": "dense", "ff": 8}), dict(att(), type="wkv2")):
        with pytest.raises(ValueError):
            rig_for(make_cfg([bad]), 1, w=ok)


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
        u = toks(40, cfg["vocab"], 1)
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


BIG = make_cfg([att(8, 2, 64, 64, 0.125, 50, 5, mlp=moe(6, 2, 96, 64, 2, (2, 1))), lat(4, 48, 16, 64, 96, 64, 0.12, 70, 1e4, mlp=moe(5, 3, 64, 160, 3, (4, 2))),
                att(4, 2, 128, 128, 0.09, 33, 20), lat(20, 16, 16, 32, 64, 112, 0.18, 40, 1e5, mlp=moe(8, 2, 128, 0, 0, None)),
                att(2, 2, 64, 128, 0.12, 16, 16), att(8, 1, 128, 64, 0.1, 100, 1), lat(3, 64, 64, 128, 64, 256, 0.08, 90, 1e6)],
               width=128, vocab=211, streams=4, loop=(0, 2, 2))


@pytest.mark.gpu
def test_gpu_matrix_core_sizes_bf16():
    """Head sizes of 64 / 128 take the matrix-core attention kernels and the vector decode kernels; long
    enough for several windows, tiles and pages per wave."""
    rig = rig_for(BIG, 6, device="cuda", dtype=torch.bfloat16, num_blocks=48)
    t = toks(150, BIG["vocab"], 4)
    want = O.forward(BIG, rig.w, t)
    ref = _bf16_ref_err(BIG, rig.w, t, want, num_blocks=48)
    for cuts in ([150], [2, 2, 3, 16, 1, 31], [100]):
        _bf16_close(rig.run_cut("a", t, cuts), want, ref)
    r32 = rig_for(BIG, 6, device="cuda", dtype=torch.float32, num_blocks=48)
    close(r32.run_cut("a", t, [70, 3]), want)


@pytest.mark.gpu
def test_gpu_large_steps_bf16():
    """1100 rows in one step: the expanded form of latent attention, the staged latent kernel, 32 query
    rows per wave, and experts on the prefill tile GEMM (widths of 256)."""
    cfg = make_cfg([lat(4, 32, 32, 64, 64, 64, 0.12, 60, 1e4, mlp=moe(3, 2, 256, 256, 1, (2, 1))),
                    att(64, 16, 64, 64, 0.12, 40, 9, mlp=moe(3, 2, 256, 256, 1, None)),
                    lat(32, 16, 16, 16, 64, 64, 0.12, 60, 1e4)], width=256, vocab=101, streams=2)
    w = O.random_weights(cfg, 7)
    rig = rig_for(cfg, w=w, device="cuda", dtype=torch.bfloat16, num_blocks=160, max_positions=2048)
    r32 = rig_for(cfg, w=w, device="cuda", dtype=torch.float32, num_blocks=160, max_positions=2048)
    t = toks(1100, cfg["vocab"], 4)
    want = r32.run_cut("a", t, [1100]).double()
    short = O.forward(cfg, w, t[:100])  # the fp32 kernels against the oracle; the rest against them
    close(want[:100].float(), short)
    ref = _row_err(rig.run_cut("a", t, [100] * 10 + [98]), want)  # portions: none of the large step's paths
    assert float(ref.quantile(0.5)) < 0.1
    _bf16_close(rig.run_cut("a", t, [1100]), want, ref)
    _bf16_close(rig.run_cut("a", t, [40, 1050]), want, ref)


@pytest.mark.gpu
def test_gpu_window_and_kept_edges():
    for dims, dtype in ((8, torch.float32), (64, torch.float32), (64, torch.bfloat16)):
        for kind in ("attention", "latent"):
            for size, keep in ((1, 0), (15, 0), (16, 3), (17, 0), (48, 16), (6, 17), (6, 65)):
                if kind == "latent" and keep:
                    continue
                layer, name = (att(2, 1, dims, dims, 0.2, size, keep), "v") if kind == "attention" else (lat(2, dims, 4, dims, 16, 16, size=size), "uv")
                cfg = make_cfg([layer], width=24, vocab=37)
                for far in sorted({keep, max(keep - 1, 0)}):
                    n = far + size + 20
                    w, t = _spiked(cfg, 11, far, n, ("l0.mix." + name,))
                    want, other = O.forward(cfg, w, t), _moved(cfg, w, t, far)
                    for cuts in ([n], [far + 1], [far + size], [2] * (n // 2 + 1)):
                        got = rig_for(cfg, w=w, device="cuda", dtype=dtype).run_cut("a", t, cuts)
                        if dtype == torch.float32:
                            close(got, want, tol=1e-4)
                        else:  # a key seen one position too long or too short moves a row by far more than this
                            assert float(_row_err(got, want).max()) < 0.04
                            assert float((want - other)[far].pow(2).mean().sqrt() / want.pow(2).mean().sqrt()) > 0.1


@pytest.mark.gpu
@pytest.mark.parametrize("dims,dtype", [(8, torch.float32), (64, torch.float32), (64, torch.bfloat16)])
def test_gpu_far_key_with_a_peaked_score(dims, dtype):
    for kind, far, size, keep in (("attention", 20, 300, 0), ("attention", 2, 40, 3), ("latent", 20, 300, 0)):
        cfg, w, t = _peaked(kind, far, 330, size, keep, dims)
        want = O.forward(cfg, w, t)
        for cuts in ([330], [310], [100, 2, 64, 130]):
            got = rig_for(cfg, w=w, num_blocks=32, device="cuda", dtype=dtype).run_cut("a", t, cuts)
            if dtype == torch.float32:
                close(got, want, tol=1e-4)
            else:
                assert float(_row_err(got, want).max()) < 0.05


@pytest.mark.gpu
def test_gpu_unequal_batch_and_reuse_fp32():
    rig = rig_for(FULL, 9, num_blocks=12, device="cuda")
    T = _plan_tokens(FULL["vocab"])
    got = _run_plans(rig, T)
    for n in T:
        close(got[n], O.forward(FULL, rig.w, T[n]))


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_gpu_stream_norm_matches_its_torch_form(dtype):
    g = torch.Generator().manual_seed(3)
    tol = 1e-5 if dtype == torch.float32 else 2e-2
    rnd = lambda *s: torch.randn(*s, generator=g)
    for T, S, d in ((5, 3, 24), (3, 4, 7), (2, 1, 1), (4, 4, 520), (3, 2, 1028), (2, 4, 2052), (2, 6, 4100), (2, 8, 8192), (1, 3, 8196), (3, 16, 301), (2, 9, 64)):
        x, y, mix, out, read, w = rnd(T, S, d), rnd(T, d), rnd(S, S), rnd(S), rnd(S), rnd(d)
        for n in (S, 1):
            for yd in (None, dtype, torch.float32):
                for rd in (read, None):
                    xc = x[:, :n].contiguous()
                    xg = xc.cuda()
                    yy = None if yd is None else y.to(yd)
                    wr = None if yd is None else (mix, out)
                    want, xw = hops.stream_norm(xc, yy, wr, rd, w, 1e-6, dtype, S)
                    cu = lambda v: v.cuda() if v is not None else None
                    got, xo = hops.stream_norm(xg, cu(yy), None if wr is None else (cu(mix), cu(out)), cu(rd), cu(w), 1e-6, dtype, S)
                    assert (xo is xg) == (xw is xc)
                    close(xo.cpu(), xw.double(), tol=1e-5)
                    close(got.cpu().float(), want.double(), tol=tol)


@pytest.mark.gpu
@pytest.mark.parametrize("E,K,groups,keep", ROUTES)
@pytest.mark.parametrize("shift", [0.0, -2.0])
def test_gpu_router_choice(E, K, groups, keep, shift):
    for d in (20, 64, 201):
        h, wr, corr = _route_case(E, d, 33, E, shift)
        ids, wts = hops.moe_router_grouped(h.cuda(), wr.cuda(), E, K, groups, keep, 1.0, soft=True, corr=corr.cuda(), best2=False, renorm=False)
        wi, ww = _route_want(h, wr, corr, K, groups, keep)
        assert torch.equal(ids.cpu(), wi)
        close(wts.cpu(), ww, tol=2e-5)
        # the sigmoid form with two best per group and renormalised weights, against the torch form
        want = hops.moe_router_grouped(h, wr, E, K, groups, keep, 1.7)
        got = hops.moe_router_grouped(h.cuda(), wr.cuda(), E, K, groups, keep, 1.7)
        assert torch.equal(got[0].cpu().sort(-1).values, want[0].sort(-1).values)
        close(got[1].cpu().sort(-1).values, want[1].double().sort(-1).values, tol=2e-5)


@pytest.mark.gpu
@pytest.mark.parametrize("E,K,groups,keep", [r for r in ROUTES if r[0] <= 16])
def test_gpu_router_choice_in_large_steps(E, K, groups, keep):
    """From 1024 rows on a workgroup takes four tokens (here also a last, partly filled one)."""
    h, wr, corr = _route_case(E, 72, 1027, E, -1.0)
    for dtype in (torch.float32, torch.bfloat16):
        hd = h.to(dtype)
        got = [hops.moe_router_grouped(hd[:n].cuda(), wr.cuda(), E, K, groups, keep, 1.3, soft=True, corr=corr.cuda(), best2=False, renorm=False)
               for n in (1027, 1000)]
        assert torch.equal(got[0][0][:1000], got[1][0])  # against the one-token workgroups
        close(got[0][1][:1000].cpu(), got[1][1].double().cpu(), tol=2e-5)
        wi, ww = _route_want(hd[1000:].float(), wr, corr, K, groups, keep)
        assert torch.equal(got[0][0][1000:].cpu(), wi)
        close(got[0][1][1000:].cpu(), ww * 1.3, tol=2e-5)
        a = hops.moe_router_grouped(hd.cuda(), wr.cuda(), E, K, groups, keep, 0.7)
        b = hops.moe_router_grouped(hd[:1000].cuda(), wr.cuda(), E, K, groups, keep, 0.7)
        assert torch.equal(a[0][:1000], b[0])
        close(a[1][:1000].cpu(), b[1].double().cpu(), tol=2e-5)


@pytest.mark.gpu
def test_gpu_router_gives_valid_experts_for_any_input():
    """Not-a-number rows still get K different experts of the list (nothing indexes by an undefined id)."""
    h = torch.randn(6, 16)
    h[2], h[4, 3] = float("nan"), float("inf")
    for E, K, groups, keep, rep in ((12, 3, 4, 2, 1), (5, 5, 1, 1, 1), (12, 3, 4, 2, 200), (5, 5, 1, 1, 200)):
        h = h.repeat(rep, 1)
        ids, _ = hops.moe_router_grouped(h.cuda(), torch.randn(E, 16).cuda(), E, K, groups, keep, 1.0, soft=True, corr=torch.randn(E).cuda(),
                                         best2=False, renorm=False)
        ids = ids.cpu()
        assert int(ids.min()) >= 0 and int(ids.max()) < E and all(len(set(r)) == K for r in ids.tolist())


@pytest.mark.gpu
@pytest.mark.parametrize("T,E,ident,K,d,ff,shared", [(5, 4, 2, 2, 24, 12, True), (33, 3, 5, 4, 64, 96, False), (1, 1, 1, 1, 32, 8, True),
                                                     (70, 6, 0, 2, 40, 36, True), (700, 3, 2, 2, 256, 256, True), (700, 5, 3, 2, 96, 64, False)])
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_gpu_squared_relu_and_identity_experts(T, E, ident, K, d, ff, shared, dtype):
    g = torch.Generator().manual_seed(6)
    rnd = lambda *s: torch.randn(*s, generator=g)
    h, w1, w2 = rnd(T, d).to(dtype), (rnd(E, ff, d) * d ** -0.5).to(dtype), (rnd(E, d, ff) * ff ** -0.5).to(dtype)
    ids = torch.stack([torch.randperm(E + ident, generator=g)[:K] for _ in range(T)]).to(torch.int32)
    wts, sh = torch.rand(T, K, generator=g), rnd(T, d).to(dtype) if shared else None
    want = torch.zeros(T, d, dtype=torch.float64)
    for t in range(T):
        for k in range(K):
            e = int(ids[t, k])
            x = h[t].double()
            want[t] += wts[t, k].double() * (x if e >= E else O.expert(x, w1[e].double(), w2[e].double()))
    if shared:
        want += sh.double()
    got = hops.moe_experts(h.cuda(), ids.cuda(), wts.cuda(), w1.cuda(), w2.cuda(), sh.cuda() if shared else None, None, act="relu_sq", identity=ident)
    close(got.cpu(), want, tol=1e-5 if dtype == torch.float32 else 3e-2)


@pytest.mark.gpu
@pytest.mark.parametrize("Hq,G,dk,dv", [(4, 2, 64, 64), (2, 1, 128, 128), (8, 1, 64, 128), (2, 2, 128, 64), (6, 2, 24, 40), (3, 3, 7, 5)])
def test_gpu_kept_window_and_gate_kernels(Hq, G, dk, dv):
    """Prompt portions and decode rows, matrix-core / vector / any-size kernels."""
    g = torch.Generator().manual_seed(8)
    n = 90
    qkv, q, k, v, kc, vc, bt, col = _keep_case(g, n, Hq, G, dk, dv)
    bt = bt.cuda()
    scale = 1.5 * dk ** -0.5
    for dtype, tol in ((torch.float32, 2e-5), (torch.bfloat16, 3e-2)):
        x, kd, vd = qkv.to(dtype), kc.to(dtype), vc.to(dtype)
        pad = torch.zeros(n, -x.shape[1] % 8, dtype=dtype)
        x = torch.cat([x, pad], -1).contiguous()
        f = x.double()
        qd = f[:, :Hq * dk].view(n, Hq, dk)
        kk = f[:, Hq * dk:Hq * dk + G * dk].view(n, G, dk)
        vv = f[:, Hq * dk + G * dk:col].view(n, G, dv)
        x, kd, vd = x.cuda(), kd.cuda(), vd.cuda()
        for size, keep in MASKS:
            want = _keep_want(qd, kk, vv, f, col, scale, size, keep)
            kw = dict(keep=keep, g_col=col)
            for a, b in ((0, 90), (5, 7), (15, 64)):
                for fast in ((0, 1) if dtype == torch.bfloat16 and dk < 64 else (0, 16, 32, 64)):
                    y = x[a:b].contiguous()
                    got = hops.window_attention_prefill(y, kd, vd, _i32(0, b - a).cuda(), _i32(a).cuda(), bt, Hq, G, dk, dv, scale, size, False,
                                                        mfma=fast, gate=y, **kw)
                    close(got.cpu().float(), want[a:b], tol=tol)
            for t in (0, 12, 16, 63, 64, 89):
                for vec in (True, False):
                    y = x[t:t + 1]
                    got = hops.window_attention_decode(y, kd, vd, bt, _i32(t + 1).cuda(), Hq, G, dk, dv, scale, size, False, vec=vec, gate=y, **kw)
                    close(got.cpu().float(), want[t:t + 1], tol=tol)


@pytest.mark.gpu
@pytest.mark.parametrize("H,R,dr", [(3, 16, 4), (16, 64, 32), (20, 128, 32), (5, 256, 64)])
def test_gpu_latent_kernels_with_a_gate(H, R, dr):
    """Every lane mapping of the latent kernels, prompts and decode rows, against the any-size kernel in fp32."""
    g = torch.Generator().manual_seed(9)
    n, pitch = 70, (R + dr + 31) // 32 * 32
    rows = torch.randn(n, pitch, generator=g).to(torch.bfloat16).float()
    rows[:, R + dr:] = 0
    kc, vc = torch.zeros(6, 16, pitch), torch.zeros(6, 1, R, 16)
    order = [2, 0, 5, 3, 1]
    for t in range(n):
        kc[order[t // 16], t % 16], vc[order[t // 16], 0, :, t % 16] = rows[t], rows[t, :R]
    qa = torch.randn(n, H, pitch, generator=g).to(torch.bfloat16).float()
    qa[..., R + dr:] = 0
    qa = qa.reshape(n, -1)
    gate = torch.randn(n, H + 5, generator=g).to(torch.bfloat16).float()
    bt, scale = _i32(*order).view(1, 5).cuda(), 1.5 * (R + dr) ** -0.5
    up = lambda t, dt: t.cuda().to(dt)
    for size in (1, 17, 40, 200):
        args32 = (up(kc, torch.float32), up(vc, torch.float32))
        args16 = (up(kc, torch.bfloat16), up(vc, torch.bfloat16))
        for a, b in ((0, n), (15, 34)):
            seg = dict(cu=_i32(0, b - a).cuda(), ctx=_i32(a).cuda(), sink=False, g_col=2)
            want = O.attend(qa[a:b].double().view(-1, H, pitch), rows[:0].double().view(0, 1, pitch), rows[:0].double().view(0, 1, pitch), scale, size) \
                if b == a else hops.latent_attention(up(qa[a:b], torch.float32), *args32, bt, H, scale, size, None, gate=up(gate[a:b], torch.float32), **seg)
            kk, vv = rows.double().view(n, 1, pitch), rows[:, :R].double().view(n, 1, R)
            full = O.attend(qa.double().view(n, H, pitch), kk, vv, scale, size) * torch.sigmoid(gate[:, 2:2 + H].double()).unsqueeze(-1)
            close(want.cpu(), full[a:b].reshape(b - a, -1), tol=2e-5)
            for split in (0, 1, 2, 4, 8, 32, 33):
                got = hops.latent_attention(up(qa[a:b], torch.bfloat16), *args16, bt, H, scale, size, None, gate=up(gate[a:b], torch.bfloat16), split=split,
                                            **seg)
                close(got.cpu().float(), full[a:b].reshape(b - a, -1), tol=3e-2)
        for t in (0, 16, 69):
            for dt, tol in ((torch.float32, 2e-5), (torch.bfloat16, 3e-2)):
                got = hops.latent_attention(up(qa[t:t + 1], dt), up(kc, dt), up(vc, dt), bt, H, scale, size, None, seq_lens=_i32(t + 1).cuda(), sink=False,
                                            gate=up(gate[t:t + 1], dt), g_col=2)
                close(got.cpu().float(), full[t:t + 1].reshape(1, -1), tol=tol)


@pytest.mark.gpu
@pytest.mark.parametrize("Hq,G,dk,dv", [(4, 2, 64, 48), (5, 1, 128, 128), (3, 3, 256, 8), (40, 8, 128, 16), (2, 2, 24, 8), (9, 3, 64, 5)])
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_gpu_head_norms_without_rotation(Hq, G, dk, dv, dtype):
    g = torch.Generator().manual_seed(10)
    n = 7
    cols = (Hq + G) * dk + G * dv
    x = (torch.randn(n, cols + (-cols % 8) + 8, generator=g) * 2).to(dtype)
    qw, kw_ = torch.randn(dk, generator=g), torch.randn(dk, generator=g)
    slots = _i32(33, 4, -1, 0, 18, 47, 20)
    res = []
    for dev in ("cpu", "cuda"):
        y = x.clone().to(dev)
        kc, vc = torch.zeros(3, 16, G * dk, dtype=dtype, device=dev), torch.zeros(3, G, dv, 16, dtype=dtype, device=dev)
        hops.rotary_cache(y, Hq, G, dk, dv, torch.arange(n, dtype=torch.int32, device=dev), hops.rotary_freq(10.0, 0, dev), False, None, kc, vc,
                          slots.to(dev), norm=1, qw=qw.to(dev), kw=kw_.to(dev), eps=1e-6)
        res.append((y.cpu(), kc.cpu(), vc.cpu()))
    q = x[:, :Hq * dk].double().view(n, Hq, dk)
    close(res[1][0][:, :Hq * dk].float(), O.rms_norm(q, qw.double(), 1e-6).reshape(n, -1), tol=1e-5 if dtype == torch.float32 else 1e-2)
    assert torch.equal(res[1][0][:, (Hq + G) * dk:], x[:, (Hq + G) * dk:])
    for a, b in zip(res[0], res[1]):
        close(b.float(), a.double(), tol=1e-5 if dtype == torch.float32 else 1e-2)


@pytest.mark.gpu
def test_gpu_greedy_generation_with_graphs():
    eng = LLMEngine(EngineConfig(model="zifisun-tiny", max_num_seqs=4, max_model_len=256, num_blocks=64,
                                 dtype="float32", max_prefill_tokens=32, mixed_prefill_tokens=16), device="cuda")
    eng.warmup()  # decode steps replay from captured hipGraphs
    cfg, w = hybrid_config_to_dict(eng.model_cfg), {k: v.cpu() for k, v in state_dict(eng.model).items()}
    prompts = [toks(n, 368, 40 + n) for n in (5, 37, 21)]
    seqs = eng.generate(prompts, SamplingParams(max_tokens=12, temperature=0.0, ignore_eos=True))
    assert eng.stats()["graph_buckets"]
    for p, s in zip(prompts, seqs):
        assert s.output_ids == O.greedy(cfg, w, p, 12)
