"""Felavik models through the framework (loader, paged cache, ragged engine, scheduler, kernels) against the
plain implementation in ``felavik_oracle`` (float64, written from the design's equations; shares no code with
the package).

Every test makes its own small configuration and random weights (checkpoint names and shapes are produced here,
saved as safetensors and read back by the package's loader).  ``dev`` runs each case on the CPU (PyTorch forms of
the ops) and, marked ``gpu``, on the HIP kernels.  Where random weights would hide a fault (a far key among
hundreds, the edge of a distance bucket, a token far back in the recurrent state), the weights are made so that one
score or one state entry stands out.
"""
import copy
import json
import math
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))
import felavik_oracle as oracle  # noqa: E402
from helpers.ragged_cases import close, portions, replay, row_err, run_mixer, step_meta, tokens  # noqa: E402

from edgellm.engine.generate import SamplingParams  # noqa: E402
from edgellm.engine.paged import PagedCache  # noqa: E402
from edgellm.engine.ragged import RaggedEngine, RaggedGenerator  # noqa: E402
from edgellm.models.configs import DecayAttnSpec, GatedAttnSpec, LayerSpec, MoESpec  # noqa: E402
from edgellm.models.registry import load_model  # noqa: E402
from edgellm.ops import seqmix  # noqa: E402

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
DEVS = ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)]
# logits error (row_err); a fault of a mechanism shows at 1e-2 and above
TOL = {"fp32": 5e-5, "bf16": 6e-2}


# --------------------------------------------------------------------------- configurations and weights
def left(heads=4, kv_heads=2, dim=8, vdim=6, buckets=8, far=20, coef=0.4, every=16, scale=None):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale if scale is not None else dim ** -0.5,
            "bias_max": far, "q_temp": {"coef": coef, "every": every}, "buckets": buckets}


def right(heads=3, dim=6, vdim=5, rot=4, base=100.0, decay=None):
    return {"heads": heads, "dim": dim, "vdim": vdim, "rot": {"dims": rot, "base": base},
            "decay": decay or [1.0 - 2.0 ** (-1 - 2 * h) for h in range(heads)]}


def parallel(l=None, r=None, left_scale=0.8, right_scale=1.3):
    return {"type": "parallel", "mixer": {"left": l or left(), "right": r or right(), "left_scale": left_scale, "right_scale": right_scale}}


def lightning(heads=3, dim=6, vdim=5, decay=None):
    return {"type": "lightning", "mixer": {"heads": heads, "dim": dim, "vdim": vdim,
                                           "decay": decay or [math.exp(-0.5 ** (2 * h + 1)) for h in range(heads)]}}


def moe(experts=6, top=2, ff=7, groups=3, keep=2):
    r = {"experts": experts, "top": top}
    if groups:
        r["groups"] = {"count": groups, "keep": keep}
    return {"kind": "moe", "router": r, "expert": {"ff": ff}}


def make_config(layers, mlps, width=20, vocab=53, eps=1e-5, scale=0.7, cap=9.0):
    """``layers`` entries may be numbers: that layer runs on the named one's weights."""
    out = []
    for l, m in zip(layers, mlps):
        out.append(dict(copy.deepcopy(out[l]), weights_of=l) if isinstance(l, int) else dict(copy.deepcopy(l), mlp=copy.deepcopy(m)))
    return {"architecture": "Felavik", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": scale},
            "logit_softcap": cap, "layers": out}


CONFIGS = {
    # both mixers, shared weights over both kinds of layer (one through another layer that shares), a layer without experts
    "shared": lambda: make_config([lightning(), parallel(), 1, lightning(heads=1, dim=9, vdim=12), 0, 2],
                                  [moe(), moe(experts=8, top=3, groups=4, keep=2), None, None, None, None]),
    # the parallel mixer first, every head its own keys, one group, one expert per token, the whole head turned
    "parallel_first": lambda: make_config([parallel(left(heads=3, kv_heads=3, dim=6, vdim=10, buckets=5, far=9, every=7),
                                                    right(heads=2, dim=8, vdim=16, rot=8), 1.0, 1.0), 0, lightning(heads=5, dim=4, vdim=8)],
                                          [moe(experts=5, top=1, groups=1, keep=1), None, None], width=24, cap=30.0),
    # odd sizes, one kv head, nothing turned, a decay that forgets at once and one that never does, all experts chosen
    "odd": lambda: make_config([parallel(left(heads=5, kv_heads=1, dim=5, vdim=3, buckets=2, far=2, coef=1.5, every=1),
                                         right(heads=2, dim=3, vdim=7, rot=0, decay=[0.0, 1.0]), -0.5, 2.0), lightning(heads=2, dim=1, vdim=3),
                                parallel(left(heads=2, kv_heads=2, dim=7, vdim=11, buckets=9, far=300), right(heads=1, dim=5, vdim=1, rot=2))],
                               [moe(experts=3, top=3, ff=5, groups=None), moe(experts=4, top=1, ff=3, groups=4, keep=1), None], width=15, scale=2.0),
}


def make_weights(cfg, seed=0):
    g = torch.Generator().manual_seed(seed)
    W = cfg["width"]
    bf = lambda t: t.to(torch.bfloat16)
    rn = lambda *s, k=1.0: bf(torch.randn(*s, generator=g) * k)
    lin = lambda o, i: rn(o, i, k=i ** -0.5)
    gain = lambda n: bf(1 + 0.2 * torch.randn(n, generator=g))
    w = {"embed": rn(cfg["vocab"], W), "head": rn(cfg["vocab"], W, k=3 * W ** -0.5), "final.norm": gain(W)}
    for i, l in enumerate(cfg["layers"]):
        if "weights_of" in l:
            continue
        p, m, M = f"l{i}.", l["mixer"], f"l{i}.mix."
        for n in ("1", "2") if l["mlp"] else ("1",):
            w[p + "norm" + n] = gain(W)

        def linear(pre, r):
            H, N, P = r["heads"], r["dim"], r["vdim"]
            w[pre + "q"], w[pre + "k"], w[pre + "v"], w[pre + "g"], w[pre + "o"] = lin(H * N, W), lin(H * N, W), lin(H * P, W), lin(H * P, W), lin(W, H * P)
        if l["type"] == "parallel":
            a, L = m["left"], M + "left."
            H, G, D, Dv = a["heads"], a["kv_heads"], a["dim"], a["vdim"]
            for n, o in (("q", H * D), ("k", G * D), ("v", G * Dv)):
                w[L + n], w[L + n + ".b"] = lin(o, W), rn(o, k=0.5)
            w[L + "q.norm"], w[L + "k.norm"], w[L + "rel"] = gain(D), gain(D), rn(a["buckets"], H)
            w[L + "g"], w[L + "o"] = lin(H * Dv, W), lin(W, H * Dv)
            linear(M + "right.", m["right"])
        else:
            linear(M, m)
            w[M + "norm"] = gain(m["heads"] * m["vdim"])
        if l["mlp"]:
            E, ff, F_ = l["mlp"]["router"]["experts"], l["mlp"]["expert"]["ff"], p + "mlp."
            w[F_ + "router"] = rn(E, W, k=2.0 * W ** -0.5)
            for k in range(E):
                w[F_ + f"e{k}.gate"], w[F_ + f"e{k}.up"], w[F_ + f"e{k}.down"] = lin(ff, W), lin(ff, W), lin(W, ff)
    return w


def as_np(w):
    return {k: v.double().numpy() for k, v in w.items()}


def save(tmp_path, cfg, w):
    from safetensors.torch import save_file
    d = tmp_path / f"m{len(os.listdir(tmp_path))}"
    d.mkdir()
    plain = copy.deepcopy(cfg)
    for l in plain["layers"]:                                # the number of distance buckets travels as a shape
        l["mixer"].get("left", {}).pop("buckets", None)
    (d / "config.json").write_text(json.dumps(plain))
    save_file({k: v.contiguous() for k, v in w.items()}, str(d / "model.safetensors"))
    return d


def load(tmp_path, cfg, w, dev, precision="fp32"):
    model, _, src = load_model(str(save(tmp_path, cfg, w)), precision=precision, device=torch.device(dev))
    assert src.startswith("checkpoint:")
    return model


def want_logits(cfg, w, toks, taps=False):
    lg, tp = oracle.forward(cfg, as_np(w), toks)
    return (torch.from_numpy(lg), torch.from_numpy(tp)) if taps else torch.from_numpy(lg)


D64 = lambda t: torch.from_numpy(np.asarray(t))
BF = lambda t: t.to(torch.bfloat16).float()


class _Spec:
    def __init__(self, **kw):
        self.__dict__.update(dict(attn=None, latent=None, delta=None, chunk_attn=None, gated_attn=None, gla=None, decay_attn=None, moe=None,
                                  ff=None), **kw)


# --------------------------------------------------------------------------- mechanisms alone
@pytest.mark.parametrize("B,far", [(2, 2), (5, 9), (8, 20), (16, 128), (32, 128), (32, 1000), (9, 5), (64, 33), (7, 40), (12, 4096), (10, 62.5)])
def test_distance_buckets(B, far):
    """Every distance up to well past the last bucket's first one; whole powers of the ratio sit on an edge."""
    rel = torch.randn(B, 3, generator=torch.Generator().manual_seed(B))
    t = seqmix.distance_bias_table(rel, far)
    want = [oracle.bucket(n, B, far) for n in range(int(2 * far))]
    assert want[0] == 0 and want[-1] == B - 1 and want == sorted(want)
    assert t.shape[1] == want.index(B - 1) + 1
    for n, b in enumerate(want):
        assert torch.equal(t[:, min(n, t.shape[1] - 1)], rel[b]), n


@pytest.mark.parametrize("dev", DEVS)
@pytest.mark.parametrize("cap", [2.5, 30.0])
def test_logit_cap(dev, cap):
    z = torch.randn(7, 1001, generator=torch.Generator().manual_seed(1)) * 3 * cap
    z[0, :3] = torch.tensor([0.0, 1e4, -1e4])
    for dt in (torch.float32, torch.bfloat16):
        x = z.to(dt)
        got = seqmix.softcap(x.to(dev), cap).cpu()
        assert got.dtype == torch.float32 and torch.allclose(got.double(), cap * torch.tanh(x.double() / cap), atol=1e-5 * cap)


@pytest.mark.parametrize("dev", DEVS)
@pytest.mark.parametrize("W", [24, 37, 1500])
def test_residual_sum_over_rows_sorted_by_expert(dev, W):
    g = torch.Generator().manual_seed(W)
    T, K = 6, 3
    x, y, parts, pw = torch.randn(T, 1, W, generator=g), torch.randn(T, W, generator=g), torch.randn(T, K, W, generator=g), torch.rand(T, K, generator=g)
    nw = torch.randn(W, generator=g)
    order = torch.randperm(T * K, generator=g)
    rows = torch.empty(T * K, dtype=torch.int32)
    rows[order] = torch.arange(T * K, dtype=torch.int32)
    D = lambda t: None if t is None else t.to(dev)
    for yy in (y, None):
        want = x.double() + (pw.double()[..., None] * parts.double()).sum(1, keepdim=True) + (0 if yy is None else yy.double()[:, None])
        for src, r in ((parts, None), (parts.view(T * K, W)[order].view(T, K, W), rows.view(T, K))):
            for nxt in (None, (None, D(nw), 1e-5)):
                X = D(x.clone())
                h = seqmix.hyper_update(X, None, None, D(yy), D(src), D(pw), nxt, D(r))
                assert torch.allclose(X.cpu().double(), want, atol=2e-5)
                if nxt:
                    assert torch.allclose(h.cpu().double(), D64(oracle.rms(want[:, 0].numpy(), 1e-5)) * nw.double(), atol=3e-5)


@pytest.mark.parametrize("dev", DEVS)
@pytest.mark.parametrize("T,E,top,groups,keep,W,ff", [(7, 6, 2, 3, 2, 20, 7), (3, 8, 3, 4, 2, 24, 16), (90, 6, 1, 1, 1, 32, 16), (130, 9, 9, 3, 3, 40, 24),
                                                      (70, 20, 4, 5, 1, 24, 8), (5, 4, 2, 2, 1, 520, 264)])
def test_silu_experts_limited_to_groups(dev, T, E, top, groups, keep, W, ff):
    """On the decode-sized and the prompt-sized expert path, added up by the residual kernel."""
    from edgellm.models.moe import MoEFeedForward
    g = torch.Generator().manual_seed(E + T)
    h = BF(torch.randn(T, W, generator=g))
    rn = lambda o, i: BF(torch.randn(o, i, generator=g) * i ** -0.5)
    w = {"router": rn(E, W)}
    for k in range(E):
        w[f"e{k}.gate"], w[f"e{k}.up"], w[f"e{k}.down"] = rn(ff, W), rn(ff, W), rn(W, ff)
    wn = as_np(w)
    mlp = {"router": {"top": top, "groups": {"count": groups, "keep": keep}}}
    m = MoEFeedForward(MoESpec(experts=E, top=top, scale=1.0, ff=ff, act="silu_glu", groups=groups, groups_keep=keep), W, torch.float32, torch.device(dev))
    m.router.copy_(w["router"]), m.w_down.copy_(torch.stack([w[f"e{k}.down"] for k in range(E)]))
    m.w_gu.copy_(torch.stack([torch.cat([w[f"e{k}.gate"], w[f"e{k}.up"]]) for k in range(E)]))
    f = m.run(h.to(dev))
    X = torch.zeros(T, 1, W, device=dev)
    seqmix.hyper_update(X, None, None, f.shared, f.parts, f.wts, None, f.rows)
    assert torch.allclose(X[:, 0].cpu().double(), D64(oracle.experts(h.double().numpy(), wn, "", mlp)), atol=5e-5)
    if keep < groups and top > keep and T > 20:               # the case tells a choice without groups apart
        free = oracle.route(h.double().numpy(), wn, "", {"top": top})[0]
        assert (free != oracle.route(h.double().numpy(), wn, "", mlp["router"])[0]).any()


ATTN_CASES = [  # left side, lengths
    (left(), (90, 13)),
    (left(heads=8, kv_heads=2, dim=16, vdim=24, buckets=32, far=100, every=64), (150, 66)),
    (left(heads=1, kv_heads=1, dim=5, vdim=3, buckets=2, far=2, every=1), (70, 3)),
    (left(heads=6, kv_heads=6, dim=7, vdim=9, buckets=9, far=33, coef=0.0), (67, 64)),
    (left(heads=6, kv_heads=1, dim=40, vdim=8, buckets=12, far=1000, every=5), (200, 97)),
]


def _attn_module(m, dev, dtype=torch.float32, W=24, seed=0):
    from edgellm.models.mixers import GatedAttention
    g = torch.Generator().manual_seed(m["dim"] + m["heads"] + seed)
    H, G, D, Dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    lin = lambda o, i: BF(torch.randn(o, i, generator=g) * i ** -0.5)
    w = {"q": lin(H * D, W), "k": lin(G * D, W), "v": lin(G * Dv, W), "g": lin(H * Dv, W), "o": lin(W, H * Dv), "rel": BF(torch.randn(m["buckets"], H, generator=g))}
    for n in "qkv":
        w[n + ".b"] = BF(0.5 * torch.randn(w[n].shape[0], generator=g))
    w["q.norm"], w["k.norm"] = (BF(1 + 0.2 * torch.randn(D, generator=g)) for _ in range(2))
    t = m["q_temp"]
    spec = GatedAttnSpec(heads=H, kv_heads=G, dim=D, vdim=Dv, scale=m["scale"], rotate_values=False, temp=False, sink=False, qkv_bias=True,
                         q_temp=(t["coef"], t["every"]), rel_buckets=m["buckets"], rel_max=m["bias_max"])
    mod = GatedAttention(spec, W, 1e-5, dtype, torch.device(dev))

    def fill():
        mod.proj_in.weight.copy_(torch.cat([w[n] for n in ("q", "k", "v", "g")])), mod.o.weight.copy_(w["o"])
        mod.qkv_b.copy_(torch.cat([w[n + ".b"] for n in "qkv"])), mod.rel.copy_(w["rel"])
        mod.q_norm.copy_(w["q.norm"]), mod.k_norm.copy_(w["k.norm"])
    fill()
    return mod, spec, w, fill, g


@pytest.mark.parametrize("dev", DEVS)
@pytest.mark.parametrize("case", ATTN_CASES)
def test_attention_alone_in_portions_and_decoding(dev, case):
    m, lens = case
    mod, spec, w, _, g = _attn_module(m, dev)
    hs = [BF(torch.randn(L, 24, generator=g)) for L in lens]
    want = [D64(oracle.attention(h.double().numpy(), as_np(w), "", m, 1e-5)) for h in hs]
    for cuts in ((5, 1, 2, 9, 1, 1, 30), (300,), (1,), (2,)):
        got, _ = run_mixer(mod, _Spec(gated_attn=spec), hs, cuts, dev)
        for g_, w_ in zip(got, want):
            assert torch.allclose(g_.double(), w_, atol=5e-5, rtol=1e-4), cuts


@pytest.mark.parametrize("dev", DEVS)
@pytest.mark.parametrize("hot", [0, 3, 5, 7, 11])
def test_bucket_edges_stand_out(dev, hot):
    """One bucket's number is far above the others, so each query reads the keys of that bucket alone: a distance on
    the wrong side of an edge shows, in prompts, portions and decoding; the table follows a change of the weights."""
    m = left(heads=3, kv_heads=1, dim=8, vdim=8, buckets=12, far=70, coef=0.1, every=30)
    mod, spec, w, fill, g = _attn_module(m, dev, seed=hot)
    h = BF(torch.randn(170, 24, generator=g))
    mod.by_distance()
    w["rel"].zero_()
    w["rel"][hot] = 30.0
    fill()
    want = D64(oracle.attention(h.double().numpy(), as_np(w), "", m, 1e-5))
    moved = dict(w, rel=torch.roll(w["rel"], 1, 0))
    assert (D64(oracle.attention(h.double().numpy(), as_np(moved), "", m, 1e-5)) - want)[80:].abs().max() > 0.1
    for cuts in ((170,), (100,) + (1,) * 70, (63, 2, 40), (9,)):
        got, _ = run_mixer(mod, _Spec(gated_attn=spec), [h], cuts, dev)
        assert torch.allclose(got[0].double(), want, atol=1e-4, rtol=1e-4), cuts


@pytest.mark.parametrize("dev", DEVS)
def test_query_temperature_steps_at_its_multiples(dev):
    """The write op alone, around the positions where floor((p + 1) / every) moves."""
    H, D, Dv, coef, every = 2, 8, 4, 0.7, 64
    T = 6
    u = torch.randn(T, 2 * D + D + Dv, generator=torch.Generator().manual_seed(0))
    cache = PagedCache([_Spec(gated_attn=GatedAttnSpec(H, 1, D, Dv, 1.0))], 40, slots=1, page=64, dtype=torch.float32, device=dev)
    s = cache.acquire()
    for start in (0, 60, 125, 2044):
        meta = step_meta(cache, {0: s}, [(0, start, T)], dev)
        q = seqmix.qk_norm_rope_write(u.to(dev), meta, None, None, 1e-5, None, None, None, cache.run(0).k, cache.run(0).v, H, 0, None, (coef, every))
        f = torch.tensor([oracle.temperature(start + t, {"coef": coef, "every": every}) for t in range(T)])
        assert f.min() < f.max() or start == 0
        assert torch.allclose(q.cpu(), u[:, :2 * D].view(T, H, D) * f[:, None, None].float(), atol=2e-6)


LINEAR_CASES = [  # heads, dim, vdim, rotated, decays, lengths
    (3, 6, 5, 4, None, (90, 13)),
    (2, 64, 64, 64, None, (200, 65)),
    (2, 33, 70, 10, [0.9, 0.999], (131, 64)),
    (1, 96, 130, 96, [0.97], (150, 30)),               # a head wider than one workgroup's columns, rotation in three tiles
    (2, 200, 96, 48, [0.5, 1.0], (140, 24)),
    (4, 16, 32, 16, [0.0, 1e-30, 1e-4, 0.3], (130, 17)),   # forgets within a token: the powers underflow
    (1, 260, 16, 32, [0.99], (70, 5)),                 # more key channels than the token-by-token kernel holds
    (5, 1, 3, 0, None, (66, 1)),
    (3, 48, 40, 32, None, (129, 70)),
]


def _linear_module(case, kind, dev, dtype=torch.float32, seed=0):
    from edgellm.models.mixers import DecayLinearAttention
    H, N, P, rot, decay, lens = case
    W = 24
    g = torch.Generator().manual_seed(N + P + seed)
    lin = lambda o, i: BF(torch.randn(o, i, generator=g) * i ** -0.5)
    w = {"q": lin(H * N, W), "k": lin(H * N, W), "v": lin(H * P, W), "g": lin(H * P, W), "o": lin(W, H * P)}
    m = {"heads": H, "dim": N, "vdim": P, "decay": decay or [1.0 - 2.0 ** (-1 - 3 * h) for h in range(H)]}
    if kind == "retention":
        m["rot"] = {"dims": rot, "base": 50.0}
        spec = DecayAttnSpec(H, N, P, tuple(m["decay"]), rot_dims=rot, rot_base=50.0, k_scale=N ** -0.5)
    else:
        w["norm"] = BF(1 + 0.2 * torch.randn(H * P, generator=g))
        spec = DecayAttnSpec(H, N, P, tuple(m["decay"]), act="silu", norm="all", gate_act="sigmoid")
    mod = DecayLinearAttention(spec, W, 1e-5, dtype, torch.device(dev))
    mod.proj_in.weight.copy_(torch.cat([w[n] for n in ("q", "k", "v", "g")])), mod.o.weight.copy_(w["o"])
    if kind == "lightning":
        mod.norm_w.copy_(w["norm"])
    return mod, spec, as_np(w), m, [BF(torch.randn(L, W, generator=g)) for L in lens]


@pytest.mark.parametrize("dev", DEVS)
@pytest.mark.parametrize("kind", ["retention", "lightning"])
@pytest.mark.parametrize("case", LINEAR_CASES)
def test_linear_attention_alone_in_portions_and_decoding(dev, kind, case):
    """Token by token, in short portions, in portions that run over 64-token chunks (also cut inside a chunk), whole:
    outputs and the state left behind, over stale state rows."""
    mod, spec, wn, m, hs = _linear_module(case, kind, dev)
    want = [D64(getattr(oracle, kind)(h.double().numpy(), wn, "", m, 1e-5)) for h in hs]
    states = [oracle.recurrence(*getattr(oracle, kind + "_inputs")(h.double().numpy(), wn, "", m), m["decay"])[1] for h in hs]
    for cuts in ((5, 1, 2, 9, 1, 1, 30), (300,), (1,), (2,), (40, 25, 3), (64,), (79, 24)):
        got, run = run_mixer(mod, _Spec(decay_attn=spec), hs, cuts, dev)
        for s, (g_, w_) in enumerate(zip(got, want)):
            assert torch.isfinite(g_).all()
            assert torch.allclose(g_.double(), w_, atol=1e-4, rtol=1e-3), cuts
            st = run.ssm[s].cpu().double()                   # slots are handed out from 0 up
            assert torch.allclose(st, D64(states[s]), atol=1e-5 * max(1.0, np.abs(states[s]).max())), cuts


@pytest.mark.parametrize("dev", DEVS)
@pytest.mark.parametrize("kind", ["retention", "lightning"])
def test_linear_attention_keeps_a_far_token(dev, kind):
    """Slow decays: one loud token 170 positions back is most of the state; it is carried across chunk and portion
    borders, and only decays that are right keep its share."""
    mod, spec, wn, m, hs = _linear_module((2, 6, 5, 4, [0.9995, 0.998], (180,)), kind, dev, seed=3)
    h = hs[0] * 0.05
    h[7] = hs[0][7] * 20
    h[177] = hs[0][177]
    want = D64(getattr(oracle, kind)(h.double().numpy(), wn, "", m, 1e-5))
    h2 = h.clone()
    h2[7] = h[8]
    assert (D64(getattr(oracle, kind)(h2.double().numpy(), wn, "", m, 1e-5)) - want)[177].abs().max() > 0.1
    for cuts in ((180,), (170,) + (1,) * 10, (64, 50, 2), (9,)):
        got, _ = run_mixer(mod, _Spec(decay_attn=spec), [h], cuts, dev)
        assert torch.allclose(got[0].double(), want, atol=1e-4, rtol=1e-3), cuts


@pytest.mark.parametrize("dev", DEVS)
@pytest.mark.parametrize("scales", [(1.0, 1.0), (0.3, -1.7), (0.0, 2.5)])
def test_both_sides_in_one_row(dev, scales):
    """The two sides with unequal sizes and scales through one input and one output projection."""
    from edgellm.models.mixers import AttentionRetention
    a, r = left(heads=3, kv_heads=1, dim=9, vdim=7), right(heads=2, dim=10, vdim=12, rot=6)
    la, spec_a, w, _, g = _attn_module(a, dev)
    W = 24
    H, N, P = r["heads"], r["dim"], r["vdim"]
    wr = {n: BF(torch.randn(o, W, generator=g) * W ** -0.5) for n, o in (("q", H * N), ("k", H * N), ("v", H * P), ("g", H * P))}
    wr["o"] = BF(torch.randn(W, H * P, generator=g) * (H * P) ** -0.5)
    spec_r = DecayAttnSpec(H, N, P, tuple(r["decay"]), rot_dims=6, rot_base=100.0, k_scale=N ** -0.5)
    mod = AttentionRetention(LayerSpec("attention_retention", gated_attn=spec_a, decay_attn=spec_r, left_scale=scales[0], right_scale=scales[1]),
                             W, 1e-5, torch.float32, torch.device(dev))
    mod.proj_in.weight.copy_(torch.cat([la.proj_in.weight.cpu()] + [wr[n] for n in ("q", "k", "v", "g")]))
    mod.o.weight.copy_(torch.cat([w["o"], wr["o"]], 1))
    for n in ("qkv_b", "rel", "q_norm", "k_norm"):
        getattr(mod.left, n).copy_(getattr(la, n))
    hs = [BF(torch.randn(L, W, generator=g)) for L in (80, 5)]
    both = {**{"left." + k: v for k, v in as_np(w).items()}, **{"right." + k: v for k, v in as_np(wr).items()}}
    m = {"left": a, "right": r, "left_scale": scales[0], "right_scale": scales[1]}
    want = [D64(oracle.parallel(h.double().numpy(), both, "", m, 1e-5)) for h in hs]
    for cuts in ((100,), (30, 1, 1), (1,)):
        got, _ = run_mixer(mod, _Spec(gated_attn=spec_a, decay_attn=spec_r), hs, cuts, dev)
        for g_, w_ in zip(got, want):
            assert torch.allclose(g_.double(), w_, atol=1e-4, rtol=1e-3), cuts


# --------------------------------------------------------------------------- whole models
@pytest.mark.parametrize("dev", DEVS)
@pytest.mark.parametrize("name", list(CONFIGS))
def test_whole_prompt_with_the_stream_after_every_layer(tmp_path, dev, name):
    cfg = CONFIGS[name]()
    w = make_weights(cfg, 1)
    toks = tokens(75, cfg["vocab"], 2)
    want, want_taps = want_logits(cfg, w, toks, taps=True)
    model = load(tmp_path, cfg, w, dev)
    eng = RaggedEngine(model, 128, slots=1, use_graphs=False)
    taps = []
    got = eng.step([("a", toks, list(range(len(toks))))], taps).cpu()
    assert len(taps) == len(cfg["layers"])
    for t, wt in zip(taps, want_taps):
        assert torch.allclose(t.cpu().double(), wt, atol=1e-4 * max(1.0, wt.abs().max().item()))
    assert close(got, want, TOL["fp32"])
    assert want.abs().max().item() > 0.5 * cfg["logit_softcap"] or name == "parallel_first"     # the cap is in reach


@pytest.mark.parametrize("dev", DEVS)
@pytest.mark.parametrize("name", list(CONFIGS))
def test_prefill_then_decode_and_portions(tmp_path, dev, name):
    cfg = CONFIGS[name]()
    w = make_weights(cfg, 3)
    toks = tokens(90, cfg["vocab"], 4)
    want = want_logits(cfg, w, toks)
    model = load(tmp_path, cfg, w, dev)
    for cuts in ([60] + [1] * 30, portions(90), [2] * 45, [1] * 90, [63, 2, 25], [64, 1, 25], [15, 2, 47, 26]):
        got, _ = replay(model, [[("a", n)] for n in cuts], {"a": toks}, 128, graphs=False)
        assert close(got["a"], want, TOL["fp32"]), cuts[:4]


@pytest.mark.parametrize("dev", DEVS)
@pytest.mark.parametrize("seed", [0, 1, 2, 3, 4])
def test_random_geometries(tmp_path, dev, seed):
    """Sizes drawn at random: heads, key / value sizes, buckets, rotated share, decays, scales, groups, layer order,
    shared weights; prompt, portions and decoding in one schedule."""
    r = np.random.RandomState(seed)
    pick = lambda *a: a[int(r.randint(0, len(a)))]
    decays = lambda H: [float(pick(0.2, 0.9, 0.99, 0.9995)) for _ in range(H)]
    layers, mlps = [], []
    for i in range(int(r.randint(2, 6))):
        G = pick(1, 2, 3)
        E, keep = G * pick(2, 3), int(r.randint(1, G + 1))
        mlps.append(pick(None, moe(E, int(r.randint(1, E // G * keep + 1)), pick(3, 8, 16), G, keep)))
        if layers and r.rand() < 0.35:
            layers.append(int(r.randint(0, i)))
            continue
        H, N = pick(1, 2, 5), pick(3, 8, 17, 40)
        if r.rand() < 0.5:
            layers.append(lightning(H, N, pick(1, 6, 16, 33), decays(H)))
        else:
            kv, B = pick(1, 2, 3), pick(2, 3, 10, 32)
            layers.append(parallel(left(kv * pick(1, 2, 4), kv, pick(3, 8, 24), pick(2, 8, 9, 40), B, B // 2 + pick(1, 5, 60, 400), pick(0.1, 1.0),
                                        pick(1, 10, 64), pick(0.1, 0.4)),
                                   right(H, N, pick(1, 6, 16, 33), pick(0, 2, N // 2 * 2), pick(20.0, 10000.0), decays(H)), pick(0.5, 1.0, 2.0), pick(0.7, -1.0)))
    cfg = make_config(layers, mlps, width=pick(12, 17, 32), vocab=41, scale=pick(0.3, 1.0, 4.0), cap=pick(5.0, 50.0))
    w = make_weights(cfg, 40 + seed)
    toks = tokens(150, cfg["vocab"], seed)
    want = want_logits(cfg, w, toks)
    model = load(tmp_path, cfg, w, dev)
    got, _ = replay(model, [[("a", n)] for n in [70, 3, 1, 1, 50, 2] + [1] * 23], {"a": toks}, 192, graphs=False)
    assert close(got["a"], want, TOL["fp32"])


@pytest.mark.parametrize("dev", DEVS)
def test_mixed_batches_reuse_pages_and_slots(tmp_path, dev):
    """Five unequal requests over six pages and three slots: portions of some beside single tokens of
    others, pages and slots of finished requests taken by later ones, a request left out of a step."""
    cfg = CONFIGS["shared"]()
    w = make_weights(cfg, 5)
    lens = {"a": 130, "b": 70, "c": 9, "d": 100, "e": 66}
    reqs = {r: tokens(n, cfg["vocab"], 30 + i) for i, (r, n) in enumerate(lens.items())}
    want = {r: want_logits(cfg, w, t) for r, t in reqs.items()}
    sched = [[("a", 60), ("b", 2), ("c", 1)], [("a", 1), ("b", 40), ("c", 3)], [("b", 1), ("c", 5)], [("a", 5)],
             [("a", 64), ("b", 27)],                         # c and b have ended: their slots and pages are free
             [("d", 63), ("e", 2)], [("d", 1), ("e", 1)], [("d", 2), ("e", 62)], [("d", 34), ("e", 1)]]
    model = load(tmp_path, cfg, w, dev)
    got, eng = replay(model, sched, reqs, 6 * 64, slots=3, graphs=False)
    for r in reqs:
        assert close(got[r], want[r], TOL["fp32"]), r
    assert eng.cache.stats()["free_pages"] == 6 and eng.cache.stats()["free_slots"] == 3
    alone, _ = replay(model, [[("d", 100)]], {"d": reqs["d"]}, 128, graphs=False)
    assert row_err(got["d"], alone["d"].double()).max().item() < 2e-5      # a batch changes nothing beyond rounding


def _far_model():
    """One attention whose key path is the negated query path without biases, and token 20 + n carries the negated
    embedding of token 10 + n: q(20 + n) = k(10 + n) while every token's score against itself is strongly negative.
    The second layer runs on the first one's weights."""
    cfg = make_config([parallel(left(heads=2, kv_heads=2, dim=32, vdim=6, far=50, scale=1.0, coef=0.2, every=50), right(heads=1), 1.5, 0.2), 0, lightning()],
                      [moe(), None, None], vocab=300, width=24)
    w = make_weights(cfg, 7)
    L = "l0.mix.left."
    w[L + "k"], w[L + "k.norm"] = -w[L + "q"], w[L + "q.norm"].clone()
    for n in "qk":
        w[L + n + ".b"].zero_()
    w["embed"][20:30] = -w["embed"][10:20]
    return cfg, w


@pytest.mark.parametrize("dev", DEVS)
@pytest.mark.parametrize("L,pairs", [(430, [(5, 429), (17, 427)]), (200, [(63, 199), (64, 198), (127, 197), (128, 196), (0, 195)])])
def test_far_keys_and_page_borders_with_sharp_scores(tmp_path, dev, L, pairs):
    """A marked key hundreds of tokens back, and marked keys at the last and first row of a page and at the
    sequence's start, found in a prompt, in portions and in decoding."""
    cfg, w = _far_model()
    toks = [40 + i % 256 for i in range(L)]
    for n, (j, i) in enumerate(pairs):
        toks[j], toks[i] = 10 + n, 20 + n
    want = want_logits(cfg, w, toks)
    probes = [i for _, i in pairs]
    other = list(toks)
    for j, _ in pairs:
        other[j] = 35
    assert row_err(want_logits(cfg, w, other)[probes], want[probes]).min().item() > 1e-2
    model = load(tmp_path, cfg, w, dev)
    for cuts in ([L], [L - 6] + [1] * 6, portions(L, mod=61)):
        got, _ = replay(model, [[("a", n)] for n in cuts], {"a": toks}, 64 * ((L + 63) // 64), graphs=False)
        assert close(got["a"][-8:], want[-8:], TOL["fp32"])


@pytest.mark.parametrize("dev", DEVS)
def test_first_tokens_of_a_sequence(tmp_path, dev):
    """Positions 0, 1, 2 alone and in every cut, in a slot that an earlier request has left."""
    cfg = CONFIGS["parallel_first"]()
    w = make_weights(cfg, 9)
    toks, before = tokens(5, cfg["vocab"], 1), tokens(30, cfg["vocab"], 2)
    want = want_logits(cfg, w, toks)
    model = load(tmp_path, cfg, w, dev)
    for cuts in ([1, 1, 1, 1, 1], [1, 4], [2, 3], [5], [3, 1, 1]):
        got, _ = replay(model, [[("z", 30)]] + [[("a", n)] for n in cuts], {"z": before, "a": toks}, 64, slots=1, graphs=False)
        assert close(got["a"], want, TOL["fp32"]), cuts


@pytest.mark.parametrize("dev", DEVS)
def test_shared_weights_keep_their_own_cache(tmp_path, dev):
    """A layer on another one's weights adds no parameters, but pages and a state of its own."""
    cfg = CONFIGS["shared"]()
    w = make_weights(cfg, 9)
    model = load(tmp_path, cfg, w, dev)
    assert model.runs == [(0, None), (1, None), (1, None), (3, None), (0, None), (1, None)]
    names = {n.split(".")[1] for n, _ in model.named_parameters() if n.startswith("layers.")}
    assert names == {"0", "1", "3"}
    cache = RaggedEngine(model, 64, slots=1).cache
    assert len(cache.runs) == 6
    for a, b in ((1, 2), (2, 5)):
        for n in ("k", "v", "ssm"):
            assert getattr(cache.run(a), n).data_ptr() != getattr(cache.run(b), n).data_ptr()
    assert cache.run(0).ssm.data_ptr() != cache.run(4).ssm.data_ptr() and cache.run(4).k is None


@pytest.mark.parametrize("dev", DEVS)
def test_bf16_model_and_long_decoding(tmp_path, dev):
    """bf16 weights and activations (fp32 stream, norms, scores, state): a prompt and 120 decoded tokens, by median
    and 90 % quantile (a near tie of two router scores can fall the other way in 16 bits)."""
    cfg = make_config([lightning(2, 16, 24), parallel(left(4, 2, 16, 24, 16, 60), right(2, 16, 32, 16)), 0, parallel(left(4, 1, 32, 32, 8, 30), right(1, 32, 16, 8)), 1],
                      [moe(8, 2, 16, 4, 2), moe(4, 1, 16, 2, 1), None, moe(6, 3, 24, 2, 1), None], width=32, vocab=64, cap=20.0)
    w = make_weights(cfg, 11)
    toks = tokens(200, cfg["vocab"], 12)
    want = want_logits(cfg, w, toks)
    model = load(tmp_path, cfg, w, dev, "bf16")
    assert model.dtype == torch.bfloat16
    got, eng = replay(model, [[("a", 80)]] + [[("a", 1)]] * 120, {"a": toks}, 256)
    e = row_err(got["a"], want)
    assert e.median().item() < 2e-2 and e.quantile(0.9).item() < TOL["bf16"], (e.median().item(), e.max().item())
    if dev == "cuda":
        assert eng.graphs_used


def _greedy_oracle(cfg, w, prompt, n):
    toks = list(prompt)
    for _ in range(n):
        lg = oracle.forward(cfg, as_np(w), toks)[0][-1]
        top = np.sort(lg)[-2:]
        if top[1] - top[0] < 1e-3:                            # a near tie is not a test of anything
            return None
        toks.append(int(np.argmax(lg)))
    return toks[len(prompt):]


@pytest.mark.parametrize("dev", DEVS)
def test_greedy_generation_through_the_scheduler(tmp_path, dev):
    """``RaggedGenerator.generate`` (scheduler, chunked prompts, fused sampler) with more prompts than slots."""
    cfg = CONFIGS["shared"]()
    w = make_weights(cfg, 13)
    prompts = [tokens(n, cfg["vocab"], 20 + n) for n in (9, 30, 5, 17)]
    model = load(tmp_path, cfg, w, dev)
    gen = RaggedGenerator(model, max_batch=2, max_seq=64, prefill_chunk=7)
    res = gen.generate(prompts, SamplingParams(max_new_tokens=6, do_sample=False, repetition_penalty=1.0), stop_at_eos=False)
    want = [_greedy_oracle(cfg, w, p, 6) for p in prompts]
    assert sum(x is not None for x in want) >= 3
    for got, x in zip(res.tokens, want):
        assert x is None or got == x


def test_checkpoint_round_trip_and_config(tmp_path):
    from edgellm.models.configs import from_hf_dir, to_felavik_config
    from edgellm.models.hf import save_hf_model
    for name in CONFIGS:
        cfg = CONFIGS[name]()
        w = make_weights(cfg, 15)
        model = load(tmp_path, cfg, w, "cpu")
        back_cfg = to_felavik_config(model.cfg)
        for k in ("embedding", "logit_softcap", "norm", "vocab", "width"):
            assert back_cfg[k] == cfg[k]
        for a, b in zip(back_cfg["layers"], cfg["layers"]):
            b["mixer"].get("left", {}).pop("buckets", None)
            if b["mlp"]:
                b["mlp"]["router"].setdefault("groups", {"count": 1, "keep": 1})
            assert a == b
        out = tmp_path / f"saved_{name}"
        save_hf_model(model, str(out))
        from safetensors.torch import load_file
        back = load_file(str(out / "model.safetensors"))
        assert set(back) == set(w)
        for k in w:
            assert back[k].shape == w[k].shape and torch.equal(back[k].float(), w[k].float()), k
        assert from_hf_dir(str(out)).layer_specs == model.cfg.layer_specs


def test_configs_that_cannot_be():
    from edgellm.models.configs import from_felavik_config
    bad = [make_config([lightning()], [m]) for m in (moe(experts=6, groups=4, keep=1), moe(experts=6, top=3, groups=3, keep=1), moe(groups=3, keep=4),
                                                     {"kind": "dense", "ff": 8})]
    bad.append(make_config([{"type": "conv", "mixer": {}}], [None]))
    bad.append(make_config([lightning(heads=2, decay=[0.5])], [None]))
    bad.append(make_config([lightning(heads=2, decay=[0.5, 1.5])], [None]))
    bad.append(make_config([parallel(left(heads=3, kv_heads=2))], [None]))
    bad.append(make_config([parallel(r=right(dim=4, rot=6))], [None]))
    bad.append(make_config([parallel(left(far=16))], [None]))                # as far as half of the (default) 32 rows
    for ref in (7, -1, 1):                                    # no such layer; itself
        c = make_config([lightning(), 0], [None, None])
        c["layers"][1]["weights_of"] = ref
        bad.append(c)
    c = make_config([lightning(), 0], [moe(), None])
    c["layers"][1]["mlp"] = None                              # differs from the layer it names
    bad.append(c)
    for c in bad:
        with pytest.raises(ValueError):
            from_felavik_config(c)


def test_evaluate_cli_runs_a_checkpoint_folder(tmp_path):
    """The evaluation command line on a checkpoint folder of this design (vocabulary wide enough for the
    byte tokenizer): loader by config.json, paged engine and scheduler, the sampling configuration, the
    confidence metric through the model's own prompt pass."""
    from edgellm.cli import evaluate
    cfg = make_config([parallel(), lightning(), 0], [moe(), moe(), None], vocab=300, width=24)
    d = save(tmp_path, cfg, make_weights(cfg, 3))
    y = tmp_path / "c.yaml"
    y.write_text(f"""
max_new_tokens: 4
temperature: 0.7
top_k: 50
top_p: 0.9
repetition_penalty: 1.1
dataset_name: sentence-transformers/natural-questions
dataset_split: train[:2]
embedder_model: "none"
models: ["{d}"]
""")
    out = evaluate.main(["--config", str(y), "--devices", "cpu", "--num_samples", "2", "--max_seq", "512",
                         "--batch_size", "2", "--prefill_chunk", "16", "--precision", "fp32"])
    assert out[str(d)]["tps"] > 0 and 0 < out[str(d)]["confidence"] <= 1


def test_trace_program_on_a_checkpoint_folder(tmp_path):
    """``bin/trace_run`` as a program: steps on standard input, logits files and ``done`` lines out."""
    cfg = CONFIGS["parallel_first"]()
    w = make_weights(cfg, 17)
    d = save(tmp_path, cfg, w)
    toks = tokens(20, cfg["vocab"], 1)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": toks[:13], "want": [0, 12]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": toks[13:15], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": toks[15:], "want": [4]}, {"id": "b", "tokens": toks[:3], "want": [2]}], "end": ["a", "b"]}]
    out = tmp_path / "out"
    r = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", str(d), "--dtype", "float32", "--out", str(out),
                        "--max-tokens", "128", "--device", "cpu"], input="\n".join(json.dumps(s) for s in steps) + "\n",
                       capture_output=True, text=True, timeout=300)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [l for l in r.stdout.splitlines() if l.startswith("done")] == ["done 0", "done 1", "done 2"]
    want = want_logits(cfg, w, toks)
    g0 = torch.from_numpy(np.fromfile(out / "0.f32", dtype="<f4").reshape(2, -1))
    g2 = torch.from_numpy(np.fromfile(out / "2.f32", dtype="<f4").reshape(2, -1))
    assert not (out / "1.f32").exists()
    assert close(g0, want[[0, 12]], TOL["fp32"]) and close(g2, torch.stack([want[19], want[2]]), TOL["fp32"])


# --------------------------------------------------------------------------- kernels only
@pytest.mark.gpu
@pytest.mark.parametrize("precision", ["fp32", "bf16"])
def test_graph_replays_against_eager_steps(tmp_path, precision):
    """Decode steps replayed from a captured graph, with eager prompt portions and synchronisations between
    the replays, against the same schedule stepped eagerly."""
    cfg = CONFIGS["shared"]()
    w = make_weights(cfg, 19)
    reqs = {"a": tokens(40, cfg["vocab"], 1), "b": tokens(32, cfg["vocab"], 2)}
    sched = [[("a", 20), ("b", 9)]] + [[("a", 1), ("b", 1)]] * 8 + [[("a", 4), ("b", 1)]] + [[("a", 1), ("b", 1)]] * 8 + \
        [[("b", 6)]]
    model = load(tmp_path, cfg, w, "cuda", precision)
    eager, _ = replay(model, sched, reqs, 256, graphs=False)
    graph, eng = replay(model, sched, reqs, 256, graphs=True)
    assert eng.graphs_used
    for r in reqs:
        assert torch.equal(eager[r], graph[r])


@pytest.mark.gpu
@pytest.mark.parametrize("kind", ["retention", "lightning"])
@pytest.mark.parametrize("case", [(2, 64, 64, 64, None, (500, 65)), (2, 40, 32, 16, [0.99, 0.9], (131, 1)), (1, 128, 128, 128, [0.999], (300, 2)),
                                  (3, 20, 136, 6, None, (100, 33))])
def test_bf16_linear_attention_in_both_forms(kind, case):
    """bf16 inputs: the chunked and the token-by-token kernels against float64 on the same rounded projections."""
    mod, spec, wn, m, hs = _linear_module(case, kind, "cuda", torch.bfloat16)
    H, N, P = spec.heads, spec.dim, spec.vdim
    g = torch.Generator().manual_seed(1)
    us = [BF(torch.randn(h.shape[0], sum(spec.in_sizes), generator=g)) for h in hs]
    eye = {n: np.eye(sum(spec.in_sizes))[a:b] for n, a, b in (("q", 0, H * N), ("k", H * N, 2 * H * N), ("v", 2 * H * N, 2 * H * N + H * P),
                                                              ("g", 2 * H * N + H * P, 2 * H * N + 2 * H * P))}
    eye.update(o=np.eye(H * P), norm=wn.get("norm"))
    want = [D64(getattr(oracle, kind)(u.double().numpy(), eye, "", m, 1e-5)) for u in us]
    for cuts in ((600,), (100, 20, 1), (7,)):
        got, _ = run_mixer(lambda u, meta, run: mod.attend(u, 0, meta, run), _Spec(decay_attn=spec), us, cuts, "cuda", torch.bfloat16)
        for a, b in zip(got, want):
            assert (a.double() - b).abs().max().item() < 1e-2 * max(1.0, b.abs().max().item()), cuts


@pytest.mark.gpu
@pytest.mark.parametrize("H,G,D,Dv,B,far", [(4, 2, 64, 64, 32, 200), (8, 2, 32, 96, 12, 1000), (6, 3, 72, 40, 8, 20), (3, 3, 128, 128, 32, 90), (4, 1, 128, 72, 6, 64),
                                            (2, 1, 48, 104, 20, 40), (5, 5, 20, 12, 8, 33), (2, 2, 136, 64, 8, 33)])
@pytest.mark.parametrize("spike", [False, True])
def test_bf16_attention_over_long_prompts(H, G, D, Dv, B, far, spike):
    """The matrix-core prompt kernel with a bias by distance (and the general kernel where it does not take the sizes),
    and decode-sized steps, against float64 on the same rounded projections; ``spike``: one far bucket stands out."""
    m = left(H, G, D, Dv, B, far, coef=0.2, every=100)
    mod, spec, w, fill, g = _attn_module(m, "cuda", torch.bfloat16)
    if spike:
        w["rel"].zero_()
        w["rel"][B - 2] = 12.0
        fill()
    n = sum(spec.proj_sizes)
    us = [BF(torch.randn(L, n, generator=g)) for L in (330, 65)]
    cut = np.cumsum((0,) + spec.proj_sizes)
    eye = as_np(w)
    for i, name in enumerate(("q", "k", "v", "g")):
        eye[name] = np.eye(n)[cut[i]:cut[i + 1]]
    want = [D64(oracle.attention_heads(u.double().numpy(), eye, "", m, 1e-5)) for u in us]
    for cuts in ((330,), (100, 1, 60), (5,)):
        got, _ = run_mixer(lambda u, meta, run: mod.attend(u, 0, meta, run), _Spec(gated_attn=spec), us, cuts, "cuda", torch.bfloat16)
        for a, b in zip(got, want):
            assert (a.double() - b).abs().max().item() < 3e-2 * max(1.0, b.abs().max().item()), cuts


@pytest.mark.gpu
@pytest.mark.parametrize("H,G,D,Dv", [(64, 8, 64, 64), (32, 16, 64, 96), (64, 16, 128, 64)])
def test_bf16_attention_with_heads_that_share_a_workgroup(H, G, D, Dv):
    """Steps large enough for two or four heads per workgroup of the matrix-core kernel, gate and scale in its
    epilogue, written beside other columns: sampled rows against float64."""
    g = torch.Generator().manual_seed(H + Dv)
    lens, dt = (3000, 1100), torch.bfloat16
    cache = PagedCache([_Spec(gated_attn=GatedAttnSpec(H, G, D, Dv, 1.0))], 70, slots=2, page=64, dtype=dt, device="cuda")
    slots = {s: cache.acquire() for s in range(2)}
    meta = step_meta(cache, slots, [(0, 0, lens[0]), (1, 0, lens[1])], "cuda")
    T = sum(lens)
    assert sum((n + 63) // 64 for n in lens) * (H // (4 if (H // G) % 4 == 0 else 2)) >= 1024
    rn = lambda *s: torch.randn(*s, generator=g).to(dt)
    u, gate, rel = rn(T, (H + G) * D + G * Dv), rn(T, H * Dv), torch.randn(H, 300, generator=g) * 2
    q = seqmix.qk_norm_rope_write(u.cuda(), meta, None, None, 1e-5, None, None, None, cache.run(0).k, cache.run(0).v, H, 0)
    wide = torch.full((T, H * Dv + 24), 7.0, dtype=dt, device="cuda")
    seqmix.window_pool_attention(q, gate.cuda(), cache.run(0).k, cache.run(0).v, None, None, meta, 0.1, None, None, None, 0, rel.cuda(),
                                 wide[:, 8:8 + H * Dv], 0.5)
    got = wide.cpu()
    assert (got[:, :8] == 7).all() and (got[:, 8 + H * Dv:] == 7).all()
    x, off = u.double(), 0
    for n in lens:
        k = x[off:off + n, H * D:(H + G) * D].view(n, G, D)
        v = x[off:off + n, (H + G) * D:].view(n, G, Dv)
        for i in (0, 63, 64, 301, 777, n - 1):
            s = torch.einsum("grd,lgd->grl", x[off + i, :H * D].view(G, H // G, D), k[:i + 1]) * 0.1
            s = s + rel.double()[:, (i - torch.arange(i + 1)).clamp(max=299)].view(G, H // G, i + 1)
            o = torch.einsum("grl,lgd->grd", torch.softmax(s, -1), v[:i + 1]).reshape(-1) * torch.sigmoid(gate[off + i].double()) * 0.5
            assert (got[off + i, 8:8 + H * Dv].double() - o).abs().max() < 2e-2 * max(1.0, o.abs().max().item()), (n, i)
        off += n


@pytest.mark.gpu
@pytest.mark.parametrize("precision", ["fp32", "bf16"])
def test_sizes_that_are_not_multiples_of_eight(tmp_path, precision):
    """Odd widths and head sizes take the scalar kernel paths and unaligned slices of the fused projections."""
    cfg = CONFIGS["odd"]()
    w = make_weights(cfg, 21)
    toks = tokens(100, cfg["vocab"], 22)
    want = want_logits(cfg, w, toks)
    model = load(tmp_path, cfg, w, "cuda", precision)
    got, _ = replay(model, [[("a", 70)], [("a", 3)]] + [[("a", 1)]] * 27, {"a": toks}, 128)
    e = row_err(got["a"], want)
    if precision == "fp32":
        assert e.max().item() < TOL["fp32"]
    else:
        assert e.median().item() < 3e-2 and e.quantile(0.9).item() < 0.1
