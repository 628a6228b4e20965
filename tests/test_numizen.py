"""Numizen models through the framework (loader, paged cache, ragged engine, scheduler, kernels) against
the plain implementation in ``numizen_oracle`` (float64, written from the design's equations; shares no
code with the package).

Every test makes its own small configuration and random weights (checkpoint names and shapes are
produced here, saved as safetensors and read back by the package's loader).  ``dev`` runs each case on
the CPU (PyTorch forms of the ops) and, marked ``gpu``, on the HIP kernels.  Where random weights would
hide a fault (a far key among hundreds, a token far back in the recurrent state), the weights are made so
that one score or one state entry stands out.
"""
import copy
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))
import numizen_oracle as oracle  # noqa: E402

from edgellm.engine.generate import SamplingParams  # noqa: E402
from edgellm.engine.paged import PagedCache  # noqa: E402
from edgellm.engine.ragged import RaggedEngine, RaggedGenerator  # noqa: E402
from edgellm.models.configs import GLASpec, LatentAttnSpec, MoESpec  # noqa: E402
from edgellm.models.registry import load_model  # noqa: E402
from edgellm.ops import seqmix  # noqa: E402

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
DEVS = ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)]
# logits error: root mean square over the vocabulary of the difference (mean taken off), over the spread of
# the oracle's logits; a fault of a mechanism shows at 1e-2 and above
TOL = {"fp32": 5e-5, "bf16": 6e-2}


# --------------------------------------------------------------------------- configurations and weights
def latent(heads=3, dim=8, rot=4, vdim=6, q_rank=10, kv_rank=12, base=100.0, scale=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank,
         "scale": scale if scale is not None else (dim + rot) ** -0.5}
    if rot:
        m["rot"] = {"dims": rot, "base": base}
    return {"type": "latent_attention", "mixer": m}


def gla(heads=3, dim=6, vdim=5, tau=8.0, rank=4):
    return {"type": "gla", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau}, "rank": rank}


def moe(experts=6, top=2, ff=7, groups=3, keep=2, shared=9):
    r = {"experts": experts, "top": top}
    if groups:
        r["groups"] = {"count": groups, "keep": keep}
    e = {"kind": "moe", "router": r, "expert": {"ff": ff}}
    if shared:
        e["shared"] = {"ff": shared}
    return e


def dense(ff=22):
    return {"kind": "dense", "ff": ff}


def make_config(layers, mlps, width=20, vocab=53, loop=None, positions=300, eps=1e-5):
    cfg = {"architecture": "Numizen", "vocab": vocab, "width": width, "max_positions": positions, "norm": {"eps": eps},
           "layers": [dict(copy.deepcopy(l), mlp=copy.deepcopy(m)) for l, m in zip(layers, mlps)]}
    if loop:
        cfg["loop"] = dict(zip(("start", "stop", "times"), loop))
    return cfg


CONFIGS = {
    # both mixers, dense and expert feed-forwards, a layer without one, a looped span in the middle
    "looped": lambda: make_config([latent(), gla(), latent(heads=2, vdim=9), gla(heads=2, dim=10, vdim=12, tau=4.0)],
                                  [dense(), moe(), None, moe(experts=8, top=3, groups=4, keep=2)], loop=(1, 3, 2)),
    # a linear-attention layer first, the loop from layer 0, one group, one expert per token, no shared expert
    "loop_first": lambda: make_config([gla(heads=1, dim=16, vdim=8, tau=16.0, rank=7), latent(heads=4, dim=6, rot=6, vdim=4, kv_rank=8)],
                                      [moe(experts=5, top=1, groups=1, keep=1, shared=0), dense(ff=9)], width=24, loop=(0, 2, 3)),
    # no loop, sizes that are odd, nothing rotated, a decay that forgets at once, all experts chosen
    "plain": lambda: make_config([latent(heads=1, dim=5, rot=0, vdim=3, q_rank=4, kv_rank=9), gla(heads=5, dim=3, vdim=7, tau=0.5, rank=1),
                                  latent(heads=5, dim=7, rot=2, vdim=11, q_rank=13, kv_rank=5)],
                                 [moe(experts=3, top=3, ff=5, groups=None, shared=2), None, dense(ff=13)], width=15),
}


def make_weights(cfg, seed=0):
    g = torch.Generator().manual_seed(seed)
    W = cfg["width"]
    bf = lambda t: t.to(torch.bfloat16)
    rn = lambda *s, k=1.0: bf(torch.randn(*s, generator=g) * k)
    lin = lambda o, i: rn(o, i, k=i ** -0.5)
    gain = lambda n: bf(1 + 0.2 * torch.randn(n, generator=g))
    w = {"embed": rn(cfg["vocab"], W), "pos": rn(cfg["max_positions"], W, k=0.4), "head": lin(cfg["vocab"], W)}

    def norm(name):
        w[name], w[name + ".b"] = gain(W), rn(W, k=0.1)
        w[name + ".alpha"] = bf(0.6 + 0.2 * torch.rand((), generator=g))
    norm("final.norm")
    for i, l in enumerate(cfg["layers"]):
        p, m, M = f"l{i}.", l["mixer"], f"l{i}.mix."
        for n in ("1", "2") if l["mlp"] else ("1",):
            norm(p + "norm" + n)
            w[p + "ls" + n] = bf(0.6 + 0.2 * torch.randn(W, generator=g))
        H, Dv = m["heads"], m["vdim"]
        if l["type"] == "gla":
            N, R = m["dim"], l["rank"]
            w[M + "q"], w[M + "k"], w[M + "v"], w[M + "g"] = lin(H * N, W), lin(H * N, W), lin(H * Dv, W), lin(H * Dv, W)
            w[M + "a1"], w[M + "a2"], w[M + "a2.b"], w[M + "norm"] = lin(R, W), lin(H * N, R), rn(H * N), gain(Dv)
        else:
            D, R, qr, kr = m["dim"], m["rot_dim"], m["q_rank"], m["kv_rank"]
            w[M + "dq"], w[M + "dq.norm"], w[M + "uq"] = lin(qr, W), gain(qr), lin(H * (D + R), qr)
            w[M + "dkv"], w[M + "dkv.norm"] = lin(kr + R, W), gain(kr)
            w[M + "uk"], w[M + "uv"], w[M + "g"] = lin(H * D, kr), lin(H * Dv, kr), lin(H * Dv, W)
        w[M + "o"] = lin(W, H * Dv)
        F_, e = p + "mlp.", l["mlp"]
        if e and e["kind"] == "moe":
            E, ff = e["router"]["experts"], e["expert"]["ff"]
            w[F_ + "router"], w[F_ + "correction"] = rn(E, W, k=2.0 * W ** -0.5), rn(E, k=0.3)
            for k in range(E):
                w[F_ + f"e{k}.up"], w[F_ + f"e{k}.down"] = lin(ff, W), lin(W, ff)
            if e.get("shared"):
                sf = e["shared"]["ff"]
                w[F_ + "shared.up"], w[F_ + "shared.down"], w[F_ + "shared.sg"] = lin(sf, W), lin(W, sf), lin(1, W)
        elif e:
            w[F_ + "gate"], w[F_ + "up"], w[F_ + "down"] = lin(e["ff"], W), lin(e["ff"], W), lin(W, e["ff"])
    return w


def as_np(w):
    return {k: v.double().numpy() for k, v in w.items()}


def save(tmp_path, cfg, w):
    from safetensors.torch import save_file
    d = tmp_path / f"m{len(os.listdir(tmp_path))}"
    d.mkdir()
    plain = dict(cfg, layers=[{k: v for k, v in l.items() if k != "rank"} for l in cfg["layers"]])   # ranks travel as shapes
    (d / "config.json").write_text(json.dumps(plain))
    save_file({k: v.contiguous() for k, v in w.items()}, str(d / "model.safetensors"))
    return d


def load(tmp_path, cfg, w, dev, precision="fp32"):
    model, _, src = load_model(str(save(tmp_path, cfg, w)), precision=precision, device=torch.device(dev))
    assert src.startswith("checkpoint:")
    return model


def tokens(n, vocab, seed):
    return torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def want_logits(cfg, w, toks, taps=False):
    lg, tp = oracle.forward(cfg, as_np(w), toks)
    return (torch.from_numpy(lg), torch.from_numpy(tp)) if taps else torch.from_numpy(lg)


def replay(model, schedule, reqs, max_tokens, slots=4, graphs=None):
    """``schedule``: steps of [(request name, token count)]; every row's logits are collected.
    A request ends (slot and pages given back) with its last token."""
    eng = RaggedEngine(model, max_tokens, slots=slots, use_graphs=graphs)
    at = {r: 0 for r in reqs}
    got = {r: [] for r in reqs}
    for step in schedule:
        entries = []
        for r, n in step:
            entries.append((r, reqs[r][at[r]:at[r] + n], list(range(n))))
            at[r] += n
        logits = eng.step(entries).cpu()
        o = 0
        for r, n in step:
            got[r].append(logits[o:o + n])
            o += n
            if at[r] == len(reqs[r]):
                eng.close(r)
    assert all(at[r] == len(reqs[r]) for r in reqs)
    return {r: torch.cat(v) for r, v in got.items()}, eng


def row_err(got, want):
    d = got.double() - want
    return (d - d.mean(-1, keepdim=True)).pow(2).mean(-1).sqrt() / want.std().item()


def close(got, want, tol):
    return row_err(got, want).max().item() < tol


def portions(total, first=2, mod=9):
    cuts, n = [], first
    while total:
        cuts.append(min(n, total))
        total -= cuts[-1]
        n = n % mod + 2
    return cuts


D64 = lambda t: torch.from_numpy(np.asarray(t))
BF = lambda t: t.to(torch.bfloat16).float()


class _Spec:
    def __init__(self, **kw):
        self.__dict__.update(dict(attn=None, latent=None, delta=None, chunk_attn=None, gated_attn=None, gla=None, moe=None, ff=None), **kw)


def run_mixer(mod, spec, hs, cuts, dev, dtype=torch.float32):
    """Interleaved sequences ``hs`` (inputs [L, W]) through a mixer alone in portions from ``cuts``, over pages
    and state rows that held something else."""
    cache = PagedCache([spec], sum((h.shape[0] + 63) // 64 for h in hs) + 1, slots=len(hs) + 1, page=64, dtype=dtype, device=dev)
    run = cache.run(0)
    for t in (run.lat, run.ssm):
        if t is not None:
            t.normal_()
    slots = {s: cache.acquire() for s in range(len(hs))}
    at, got, step_i = [0] * len(hs), [[] for _ in hs], 0
    while any(at[s] < hs[s].shape[0] for s in range(len(hs))):
        step = [(s, at[s], min(cuts[(step_i + s) % len(cuts)], hs[s].shape[0] - at[s])) for s in range(len(hs)) if at[s] < hs[s].shape[0]]
        for s, st, n in step:
            cache.extend(slots[s], st + n)
        meta = seqmix.RaggedMeta.build([(slots[s], st, n) for s, st, n in step], cache.page_table, cache.page, dev)
        with torch.no_grad():
            out = mod(torch.cat([hs[s][st:st + n] for s, st, n in step]).to(dev, dtype), meta, run).float().cpu()
        o = 0
        for s, st, n in step:
            got[s].append(out[o:o + n])
            o += n
            at[s] += n
        step_i += 1
    return [torch.cat(g) for g in got], run


# --------------------------------------------------------------------------- mechanisms alone
@pytest.mark.parametrize("dev", DEVS)
@pytest.mark.parametrize("W", [24, 37, 300, 1500])
def test_residual_sum_with_the_next_norms(dev, W):
    torch.manual_seed(W)
    T, K = 6, 3
    x, m, y, parts = torch.randn(T, W), torch.randn(T, W), torch.randn(T, W), torch.randn(T, K, W)
    s1, s2, yw, pw = torch.randn(W), torch.randn(W), torch.rand(T), torch.rand(T, K)
    order = torch.randperm(T * K)
    rows = torch.empty(T * K, dtype=torch.int32)
    rows[order] = torch.arange(T * K, dtype=torch.int32)
    sorted_parts = parts.view(T * K, W)[order].view(T, K, W)
    norms = [(torch.randn(W), torch.randn(W), torch.rand(1) + 0.5) for _ in range(2)]
    D = lambda t: None if t is None else t.to(dev)
    mix = (pw.double()[..., None] * parts.double()).sum(1)
    cases = [  # m, m_scale, y, y_w, parts, part_w, rows, f_scale -> what joins the stream
        ((m, s1, y, yw, parts, pw, None, s2), m.double() * s1 + (yw.double()[:, None] * y + mix) * s2),
        ((m, s1, y, yw, sorted_parts, pw, rows.view(T, K), s2), m.double() * s1 + (yw.double()[:, None] * y + mix) * s2),
        ((m, None, y, None, None, None, None, None), m.double() + y),
        ((m, s1, None, None, parts, pw, None, s2), m.double() * s1 + mix * s2),
        ((m, s1, None, None, None, None, None, None), m.double() * s1),
        ((None,) * 8, torch.zeros(T, W, dtype=torch.float64))]
    for args, add in cases:
        want = x.double() + add
        for nn in (0, 1, 2):
            xd = D(x.clone())
            h = seqmix.parallel_update(xd, tuple(tuple(D(t) for t in n) for n in norms[:nn]), torch.float32, *[D(a) for a in args])
            assert len(h) == nn and torch.allclose(xd.cpu().double(), want, atol=2e-5)
            for got, (w, b, al) in zip(h, norms):
                ref = D64(oracle.dynamic_tanh(want.numpy(), {"n": w.double().numpy(), "n.b": b.double().numpy(), "n.alpha": al.double().item()}, "n"))
                assert torch.allclose(got.cpu().double(), ref, atol=3e-5)


@pytest.mark.parametrize("dev", DEVS)
@pytest.mark.parametrize("ff", [7, 64, 300, 2056])
def test_gelu_gated_unit(dev, ff):
    torch.manual_seed(ff)
    u = torch.randn(5, 2 * ff + 8) * 3
    u[0, :4] = torch.tensor([-60.0, 60.0, -9.0, 0.0])
    want = D64(oracle.gelu_tanh(u[:, :ff].double().numpy())) * u[:, ff:2 * ff].double()
    assert torch.allclose(seqmix.glu_gelu(u.to(dev), ff).cpu().double(), want, atol=2e-5, rtol=2e-6)


@pytest.mark.parametrize("dev", DEVS)
def test_embedding_with_learned_positions(dev):
    torch.manual_seed(0)
    table, pos = torch.randn(11, 300), torch.randn(70, 300)
    ids = torch.tensor([3, 10, 0, 7, 7])
    cache = PagedCache([], 4, slots=2, page=64, device=dev)
    a, b = cache.acquire(), cache.acquire()
    meta = seqmix.RaggedMeta.build([(a, 0, 2), (b, 67, 3)], cache.page_table, 64, dev)
    got = seqmix.embedding_learned(ids.to(dev), meta, table.to(dev), pos.to(dev)).cpu()
    assert torch.allclose(got, table[ids] + pos[[0, 1, 67, 68, 69]])


ROUTES = [  # experts, top, groups, keep, spread of the correction
    (6, 2, 3, 2, 0.3), (20, 4, 5, 3, 0.05), (70, 5, 7, 1, 0.5), (8, 3, 1, 1, 0.2), (9, 9, 3, 3, 1.0), (130, 1, 65, 2, 2.0), (12, 6, 2, 1, 0.0)]


@pytest.mark.parametrize("dev", DEVS)
@pytest.mark.parametrize("E,top,groups,keep,spread", ROUTES)
def test_router_corrected_and_limited_to_groups(dev, E, top, groups, keep, spread):
    """Choice by score + correction inside the kept groups (the correction may make every choice score
    negative), weights by the score alone; the shared expert's gate from the last row."""
    g = torch.Generator().manual_seed(E + top)
    T, W = 40, 24
    h, router = torch.randn(T, W, generator=g), torch.randn(E, W, generator=g) * 0.4
    corr, sg = torch.randn(E, generator=g) * spread - (2.0 if spread > 0.4 else 0.0), torch.randn(1, W, generator=g)
    w = {"router": router.double().numpy(), "correction": corr.double().numpy()}
    idx, wt = oracle.route(h.double().numpy(), w, "", {"top": top, "groups": {"count": groups, "keep": keep}})
    gi, gw, gate = seqmix.moe_route_grouped(h.to(dev), torch.cat([router, sg]).to(dev), top, 1.0, corr.to(dev), groups, keep, True)
    assert np.array_equal(gi.cpu().numpy(), idx)
    assert torch.allclose(gw.cpu().double(), D64(wt), atol=2e-6)
    assert torch.allclose(gate.cpu().double(), torch.sigmoid(h.double() @ sg.double().t())[:, 0], atol=1e-6)
    gi, gw, gate = seqmix.moe_route_grouped(h.to(dev), router.to(dev), top, 2.0, None, groups, keep)
    idx, wt = oracle.route(h.double().numpy(), {"router": w["router"]}, "", {"top": top, "groups": {"count": groups, "keep": keep}})
    assert gate is None and np.array_equal(gi.cpu().numpy(), idx) and torch.allclose(gw.cpu().double(), 2 * D64(wt), atol=4e-6)
    if keep < groups and top > keep:                          # the case tells a choice without groups apart
        free = oracle.route(h.double().numpy(), w, "", {"top": top})[0]
        limited = oracle.route(h.double().numpy(), w, "", {"top": top, "groups": {"count": groups, "keep": keep}})[0]
        assert (free != limited).any()


@pytest.mark.parametrize("dev", DEVS)
@pytest.mark.parametrize("T,E,top,W,ff,sff", [(7, 6, 2, 20, 7, 9), (3, 8, 3, 24, 16, 40), (90, 6, 1, 32, 16, 0), (130, 9, 9, 40, 24, 8),
                                              (5, 4, 2, 520, 264, 1032)])
def test_squared_relu_experts_with_a_gated_shared_expert(dev, T, E, top, W, ff, sff):
    """On the decode-sized and the prompt-sized expert path, added up by the residual kernel."""
    from edgellm.models.moe import MoEFeedForward
    torch.manual_seed(E)
    h = BF(torch.randn(T, W))
    w = {"router": BF(torch.randn(E, W) * W ** -0.5), "correction": BF(torch.randn(E) * 0.2)}
    for k in range(E):
        w[f"e{k}.up"], w[f"e{k}.down"] = BF(torch.randn(ff, W) * W ** -0.5), BF(torch.randn(W, ff) * ff ** -0.5)
    mlp = {"router": {"top": top, "groups": {"count": 1, "keep": 1}}}
    if sff:
        mlp["shared"] = {"ff": sff}
        w["shared.up"], w["shared.down"], w["shared.sg"] = BF(torch.randn(sff, W) * W ** -0.5), BF(torch.randn(W, sff) * sff ** -0.5), \
            BF(torch.randn(1, W) * W ** -0.5)
    want = D64(oracle.moe_ff(h.double().numpy(), {k: v.double().numpy() for k, v in w.items()}, "", mlp))
    spec = MoESpec(experts=E, top=top, scale=1.0, ff=ff, shared_ff=sff, router="softmax", act="relu2", correction=True, shared_gate=bool(sff))
    m = MoEFeedForward(spec, W, torch.float32, torch.device(dev))
    m.router.copy_(torch.cat([w["router"]] + ([w["shared.sg"]] if sff else []))), m.correction.copy_(w["correction"])
    m.w_gu.copy_(torch.stack([w[f"e{k}.up"] for k in range(E)])), m.w_down.copy_(torch.stack([w[f"e{k}.down"] for k in range(E)]))
    if sff:
        m.shared_gu.weight.copy_(w["shared.up"]), m.shared_down.weight.copy_(w["shared.down"])
    x = torch.zeros(T, W, device=dev)
    f = m.run(h.to(dev))
    seqmix.parallel_update(x, (), torch.float32, None, None, f.shared, f.shared_w, f.parts, f.wts, f.rows)
    assert torch.allclose(x.cpu().double(), want, atol=5e-5)
    plain = seqmix.moe_experts(h.to(dev), seqmix.moe_route_grouped(h.to(dev), m.router, top, 1.0, m.correction, gate=bool(sff))[0],
                               m.w_gu, m.w_down, 0.0, "relu2").cpu()                       # in (token, choice) order
    idx = oracle.route(h.double().numpy(), {k: v.double().numpy() for k, v in w.items()}, "", {"top": top})[0]
    t, k = T - 1, top - 1
    e = idx[t, k]
    ref = D64(oracle.relu2(h[t].double().numpy() @ w[f"e{e}.up"].double().numpy().T) @ w[f"e{e}.down"].double().numpy().T)
    assert torch.allclose(plain[t, k].double(), ref, atol=5e-5)


LATENT_CASES = [  # heads, dim, rot, vdim, q rank, kv rank, gate, lengths
    (3, 8, 4, 6, 10, 12, True, (90, 13)),
    (4, 16, 8, 16, 24, 32, True, (150, 66)),
    (1, 5, 0, 3, 4, 9, False, (70, 3)),                 # nothing rotated, odd sizes, no gate
    (5, 7, 2, 11, 13, 5, True, (67, 64)),
    (2, 40, 32, 24, 16, 96, True, (200, 97)),
]


@pytest.mark.parametrize("dev", DEVS)
@pytest.mark.parametrize("case", LATENT_CASES)
def test_gated_latent_attention_alone_in_portions_and_decoding(dev, case):
    from edgellm.models.mixers import LatentAttention
    H, D, R, Dv, qr, kr, gate, lens = case
    W = 24
    g = torch.Generator().manual_seed(D + H)
    lin = lambda o, i: BF(torch.randn(o, i, generator=g) * i ** -0.5)
    gain = lambda n: BF(1 + 0.2 * torch.randn(n, generator=g))
    m = latent(H, D, R, Dv, qr, kr, scale=1.5 * (D + R) ** -0.5)["mixer"]
    w = {"dq": lin(qr, W), "dq.norm": gain(qr), "uq": lin(H * (D + R), qr), "dkv": lin(kr + R, W), "dkv.norm": gain(kr), "uk": lin(H * D, kr),
         "uv": lin(H * Dv, kr), "o": lin(W, H * Dv)}
    if gate:
        w["g"] = lin(H * Dv, W)
    hs = [BF(torch.randn(L, W, generator=g)) for L in lens]
    wn = {k: v.double().numpy() for k, v in w.items()}
    want = [D64(oracle.latent_attention(h.double().numpy(), wn, "", m, 1e-5)) for h in hs]
    spec = LatentAttnSpec(heads=H, dim=D, rot_dim=R, vdim=Dv, q_rank=qr, kv_rank=kr, scale=m["scale"], rot_dims=R, rot_base=100.0, gate=gate)
    mod = LatentAttention(spec, W, 1e-5, torch.float32, torch.device(dev))
    mod.proj_in.weight.copy_(torch.cat([w["dq"], w["dkv"]] + ([w["g"]] if gate else [])))
    mod.q_norm.copy_(w["dq.norm"]), mod.kv_norm.copy_(w["dkv.norm"]), mod.uq.weight.copy_(w["uq"]), mod.o.weight.copy_(w["o"])
    mod.uk.copy_(w["uk"].view(H, D, kr)), mod.uv.copy_(w["uv"].view(H, Dv, kr).transpose(1, 2))
    for cuts in ((5, 1, 2, 9, 1, 1, 30), (300,), (1,), (2,)):
        got, _ = run_mixer(mod, _Spec(latent=spec), hs, cuts, dev)
        for g_, w_ in zip(got, want):
            assert torch.allclose(g_.double(), w_, atol=5e-5, rtol=1e-4)


GLA_CASES = [  # heads, dim, vdim, tau, rank, decay bias, lengths
    (3, 6, 5, 8.0, 4, 0.0, (90, 13)),
    (2, 64, 64, 16.0, 16, 1.0, (200, 65)),
    (2, 33, 70, 4.0, 3, 2.0, (131, 64)),
    (1, 100, 130, 16.0, 16, 3.0, (150, 30)),           # a head wider than one workgroup's columns
    (2, 200, 96, 2.0, 8, 4.0, (140, 24)),
    (4, 16, 32, 0.25, 37, -4.0, (130, 17)),            # forgets within a token: the state underflows
    (2, 40, 24, 1.0, 2, -12.0, (129, 70)),             # a 16-token block decays by far more than fp32's range
    (1, 260, 16, 16.0, 4, 2.0, (70, 5)),               # more key channels than the token-by-token kernel holds
]


def _gla_module(case, dev, dtype=torch.float32, seed=0):
    from edgellm.models.mixers import GatedLinearAttention
    H, N, P, tau, R, bias, lens = case
    W = 24
    g = torch.Generator().manual_seed(N + P + seed)
    lin = lambda o, i: BF(torch.randn(o, i, generator=g) * i ** -0.5)
    w = {"q": lin(H * N, W), "k": lin(H * N, W), "v": lin(H * P, W), "g": lin(H * P, W), "a1": lin(R, W), "a2": BF(torch.randn(H * N, R, generator=g)),
         "a2.b": BF(bias + torch.randn(H * N, generator=g)), "norm": BF(1 + 0.2 * torch.randn(P, generator=g)), "o": lin(W, H * P)}
    spec = GLASpec(heads=H, dim=N, vdim=P, tau=tau, decay_rank=R)
    mod = GatedLinearAttention(spec, W, 1e-5, dtype, torch.device(dev))
    mod.proj_in.weight.copy_(torch.cat([w[n] for n in ("q", "k", "v", "g", "a1")]))
    mod.a2.copy_(w["a2"]), mod.a2_b.copy_(w["a2.b"]), mod.norm_w.copy_(w["norm"]), mod.o.weight.copy_(w["o"])
    hs = [BF(torch.randn(L, W, generator=g)) for L in lens]
    return mod, spec, {k: v.double().numpy() for k, v in w.items()}, hs


@pytest.mark.parametrize("dev", DEVS)
@pytest.mark.parametrize("case", GLA_CASES)
def test_gated_linear_attention_alone_in_portions_and_decoding(dev, case):
    """Token by token, in short portions, in portions that run over 64-token chunks (also cut inside a chunk and
    inside a 16-token block), whole: outputs and the state left behind, over stale state rows."""
    mod, spec, wn, hs = _gla_module(case, dev)
    m = {"heads": spec.heads, "dim": spec.dim, "vdim": spec.vdim, "tau": spec.tau}
    want = [D64(oracle.gla(h.double().numpy(), wn, "", m, 1e-5)) for h in hs]
    states = []
    for h in hs:
        x = h.double().numpy()
        L = x.shape[0]
        k, v = (x @ wn["k"].T).reshape(L, spec.heads, spec.dim), (x @ wn["v"].T).reshape(L, spec.heads, spec.vdim)
        states.append(oracle.gla_recurrence(k, k, v, oracle.gla_decays(x, wn, "", m))[1])
    for cuts in ((5, 1, 2, 9, 1, 1, 30), (300,), (1,), (2,), (40, 25, 3), (64,), (79, 24)):
        got, run = run_mixer(mod, _Spec(gla=spec), hs, cuts, dev)
        for s, (g_, w_) in enumerate(zip(got, want)):
            assert torch.isfinite(g_).all()
            # a head's output is divided by its own root mean square: where that is far below the state's size the
            # norm magnifies rounding, so the bound is relative to the row as well
            assert torch.allclose(g_.double(), w_, atol=1e-4, rtol=1e-3), cuts
        for s in range(len(hs)):                              # slots are handed out from 0 up
            st = run.ssm[s].cpu().double()
            assert torch.allclose(st, D64(states[s]), atol=1e-5 * max(1.0, np.abs(states[s]).max())), cuts


@pytest.mark.parametrize("dev", DEVS)
def test_linear_attention_keeps_a_far_token(dev):
    """Slow decays: one planted key / value pair 170 tokens back dominates the read of a matching query; the state
    carries it across chunk and portion borders."""
    case = (2, 5, 6, 16.0, 4, 9.0, (180,))
    mod, spec, wn, hs = _gla_module(case, dev, seed=3)
    wn["k"] = wn["q"].copy()
    mod.proj_in.weight[10:20].copy_(mod.proj_in.weight[:10])
    h = hs[0] * 0.05
    rng = np.random.RandomState(9)
    null = lambda a: np.linalg.svd(a)[2][a.shape[0]:]
    query = rng.randn(12) @ null(wn["v"])                     # no value of its own
    h[177] = torch.from_numpy(4 * query).float()
    h[7] = h[177] + torch.from_numpy(4 * rng.randn(14) @ null(wn["k"])).float()    # the query's key, another value
    m = {"heads": 2, "dim": 5, "vdim": 6, "tau": 16.0}
    want = D64(oracle.gla(h.double().numpy(), wn, "", m, 1e-5))
    h2 = h.clone()
    h2[7] = h[8]
    assert (D64(oracle.gla(h2.double().numpy(), wn, "", m, 1e-5)) - want)[177].abs().max() > 0.1
    for cuts in ((180,), (170,) + (1,) * 10, (64, 50, 2), (9,)):
        got, _ = run_mixer(mod, _Spec(gla=spec), [h], cuts, dev)
        assert torch.allclose(got[0].double(), want, atol=1e-4, rtol=1e-3), cuts


# --------------------------------------------------------------------------- whole models
@pytest.mark.parametrize("dev", DEVS)
@pytest.mark.parametrize("name", list(CONFIGS))
def test_whole_prompt_with_the_stream_after_every_run(tmp_path, dev, name):
    cfg = CONFIGS[name]()
    w = make_weights(cfg, 1)
    toks = tokens(75, cfg["vocab"], 2)
    want, want_taps = want_logits(cfg, w, toks, taps=True)
    model = load(tmp_path, cfg, w, dev)
    eng = RaggedEngine(model, 128, slots=1, use_graphs=False)
    taps = []
    got = eng.step([("a", toks, list(range(len(toks))))], taps).cpu()
    assert len(taps) == len(oracle.run_order(cfg))
    for t, wt in zip(taps, want_taps):
        assert torch.allclose(t.cpu().double(), wt, atol=1e-4 * max(1.0, wt.abs().max().item()))
    assert close(got, want, TOL["fp32"])


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
@pytest.mark.parametrize("seed", [0, 1, 2, 3])
def test_random_geometries(tmp_path, dev, seed):
    """Sizes drawn at random: heads, key / value sizes, ranks, rotated share, decay constants, groups, loops;
    prompt, portions and decoding in one schedule."""
    r = np.random.RandomState(seed)
    layers, mlps = [], []
    for _ in range(int(r.randint(2, 5))):
        if r.rand() < 0.5:
            layers.append(gla(heads=int(r.choice([1, 2, 5])), dim=int(r.choice([3, 8, 17, 40])), vdim=int(r.choice([1, 6, 16, 33])),
                              tau=float(r.choice([0.5, 1.0, 7.0, 16.0])), rank=int(r.choice([1, 4, 9]))))
        else:
            layers.append(latent(heads=int(r.choice([1, 2, 5])), dim=int(r.choice([3, 8, 12])), rot=int(r.choice([0, 2, 6])),
                                 vdim=int(r.choice([2, 8, 9])), q_rank=int(r.choice([3, 8, 14])), kv_rank=int(r.choice([4, 8, 11])),
                                 base=float(r.choice([50.0, 10000.0]))))
        G = int(r.choice([1, 2, 3]))
        E, keep = G * int(r.choice([2, 3])), int(r.randint(1, G + 1))
        mlps.append([None, dense(int(r.choice([5, 16, 33]))), moe(E, int(r.randint(1, E // G * keep + 1)), int(r.choice([3, 8])), G, keep,
                                                                  int(r.choice([0, 5, 16])))][int(r.randint(0, 3))])
    n = len(layers)
    start = int(r.randint(0, n))
    loop = (start, int(r.randint(start + 1, n + 1)), int(r.choice([1, 2, 3]))) if r.rand() < 0.7 else None
    cfg = make_config(layers, mlps, width=int(r.choice([12, 17, 32])), vocab=41, loop=loop, positions=151)
    w = make_weights(cfg, 40 + seed)
    toks = tokens(150, cfg["vocab"], seed)
    want = want_logits(cfg, w, toks)
    model = load(tmp_path, cfg, w, dev)
    cuts = [70, 3, 1, 1, 50, 2] + [1] * 23
    got, _ = replay(model, [[("a", n)] for n in cuts], {"a": toks}, 192, graphs=False)
    assert close(got["a"], want, TOL["fp32"])


@pytest.mark.parametrize("dev", DEVS)
def test_mixed_batches_reuse_pages_and_slots(tmp_path, dev):
    """Five unequal requests over six pages and three slots: portions of some beside single tokens of
    others, pages and slots of finished requests taken by later ones, a request left out of a step."""
    cfg = CONFIGS["looped"]()
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
    """One latent-attention layer whose query and key paths share their matrices with a large scale and no
    positions: the key path is the negated query path and token 20 + n carries the negated embedding of token
    10 + n, so q(20 + n) = k(10 + n) while every token's score against itself is strongly negative (the first
    norm has no bias, which makes it odd)."""
    cfg = make_config([latent(heads=2, dim=32, rot=2, vdim=6, q_rank=10, kv_rank=10, scale=2.0), gla()], [None, dense()], vocab=300, width=24,
                      positions=500)
    w = make_weights(cfg, 7)
    M = "l0.mix."
    w["pos"].zero_(), w["l0.norm1.b"].zero_()
    uq = w[M + "uq"].view(2, 34, 10)
    w[M + "dkv"] = torch.cat([w[M + "dq"], torch.zeros_like(w[M + "dkv"][10:])])
    w[M + "dkv.norm"], w[M + "uk"] = w[M + "dq.norm"].clone(), -uq[:, :32].reshape(64, 10).contiguous()
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
    cfg = CONFIGS["loop_first"]()
    w = make_weights(cfg, 9)
    toks, before = tokens(5, cfg["vocab"], 1), tokens(30, cfg["vocab"], 2)
    want = want_logits(cfg, w, toks)
    model = load(tmp_path, cfg, w, dev)
    for cuts in ([1, 1, 1, 1, 1], [1, 4], [2, 3], [5], [3, 1, 1]):
        got, _ = replay(model, [[("z", 30)]] + [[("a", n)] for n in cuts], {"z": before, "a": toks}, 64, slots=1, graphs=False)
        assert close(got["a"], want, TOL["fp32"]), cuts


@pytest.mark.parametrize("dev", DEVS)
def test_no_sequence_outgrows_the_position_table(tmp_path, dev):
    cfg = make_config([latent(), gla()], [dense(), None], positions=20)
    w = make_weights(cfg, 10)
    toks = tokens(20, cfg["vocab"], 1)
    model = load(tmp_path, cfg, w, dev)
    eng = RaggedEngine(model, 256, slots=2, use_graphs=False)
    got = eng.step([("a", toks, list(range(20)))]).cpu()
    assert close(got, want_logits(cfg, w, toks), TOL["fp32"])
    with pytest.raises(ValueError, match="positions"):
        eng.step([("a", [1], [0])])
    with pytest.raises(ValueError, match="positions"):
        eng.step([("b", [1] * 21, [0])])
    assert eng.length("a") == 20 and "b" not in eng.live      # a refused step changes nothing
    gen = RaggedGenerator(model, max_batch=1, max_seq=256)
    assert gen.max_seq == 20
    sched = gen.slot_decoder(SamplingParams(max_new_tokens=6))
    assert sched.can_admit(14, 6) and not sched.can_admit(15, 6)


@pytest.mark.parametrize("dev", DEVS)
def test_bf16_model_and_long_decoding(tmp_path, dev):
    """bf16 weights and activations (fp32 stream, norms, scores, state): a prompt and 120 decoded tokens, by median
    and 90 % quantile (a near tie of two router scores can fall the other way in 16 bits)."""
    cfg = make_config([latent(heads=2, dim=16, rot=8, vdim=16, q_rank=16, kv_rank=24), gla(heads=2, dim=16, vdim=24, tau=16.0),
                       latent(heads=4, dim=32, rot=32, vdim=32, q_rank=32, kv_rank=96)], [moe(8, 2, 16, 4, 2, 24), moe(4, 1, 16, 2, 1, 8), dense(48)],
                      width=32, vocab=64, loop=(0, 2, 2))
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
    cfg = CONFIGS["looped"]()
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
    from edgellm.models.configs import from_hf_dir, to_numizen_config
    from edgellm.models.hf import save_hf_model
    for name in CONFIGS:
        cfg = CONFIGS[name]()
        w = make_weights(cfg, 15)
        model = load(tmp_path, cfg, w, "cpu")
        back_cfg = to_numizen_config(model.cfg)
        assert back_cfg.get("loop") == cfg.get("loop") and back_cfg["max_positions"] == cfg["max_positions"]
        for a, b in zip(back_cfg["layers"], cfg["layers"]):
            assert a["type"] == b["type"] and a["mixer"] == b["mixer"]
            if b["mlp"] and b["mlp"]["kind"] == "moe":
                b["mlp"]["router"].setdefault("groups", {"count": 1, "keep": 1})
            assert a["mlp"] == b["mlp"]
        out = tmp_path / f"saved_{name}"
        save_hf_model(model, str(out))
        from safetensors.torch import load_file
        back = load_file(str(out / "model.safetensors"))
        assert set(back) == set(w)
        for k in w:
            assert back[k].shape == w[k].shape and torch.equal(back[k].float(), w[k].float()), k
        assert from_hf_dir(str(out)).layer_specs == model.cfg.layer_specs


def test_configs_that_cannot_be(tmp_path):
    from edgellm.models.configs import from_numizen_config
    for mlp in (moe(experts=6, groups=4, keep=1), moe(experts=6, top=3, groups=3, keep=1), moe(experts=6, groups=3, keep=4)):
        with pytest.raises(ValueError):
            from_numizen_config(make_config([gla()], [mlp]))
    with pytest.raises(ValueError):
        from_numizen_config(make_config([gla(), gla()], [None, None], loop=(1, 1, 2)))
    with pytest.raises(ValueError):
        from_numizen_config(make_config([{"type": "conv", "mixer": {}}], [None]))


def test_evaluate_cli_runs_a_checkpoint_folder(tmp_path):
    """The evaluation command line on a checkpoint folder of this design (vocabulary wide enough for the
    byte tokenizer): loader by config.json, paged engine and scheduler, the sampling configuration, the
    confidence metric through the model's own prompt pass."""
    from edgellm.cli import evaluate
    cfg = make_config([latent(), gla()], [dense(), moe()], vocab=300, width=24, positions=256)
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
    cfg = CONFIGS["loop_first"]()
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
    cfg = CONFIGS["looped"]()
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
@pytest.mark.parametrize("case", [(2, 64, 64, 16.0, 16, 1.0, (500, 65)), (2, 40, 32, 4.0, 8, 2.0, (131, 1)), (1, 128, 128, 16.0, 16, 3.0, (300, 2)),
                                  (3, 20, 136, 1.0, 4, 0.0, (100, 33))])
def test_bf16_linear_attention_in_both_forms(case):
    """bf16 inputs: the chunked and the token-by-token kernels against float64 on the same rounded projections."""
    mod, spec, wn, hs = _gla_module(case, "cuda", torch.bfloat16)
    H, N, P = spec.heads, spec.dim, spec.vdim
    g = torch.Generator().manual_seed(1)
    us = [BF(torch.randn(h.shape[0], sum(spec.in_sizes), generator=g)) for h in hs]
    want = []
    for u in us:
        x, L = u.double().numpy(), u.shape[0]
        z = x[:, 2 * H * N + 2 * H * P:] @ wn["a2"].T + wn["a2.b"]
        o, _ = oracle.gla_recurrence(x[:, :H * N].reshape(L, H, N) * N ** -0.5, x[:, H * N:2 * H * N].reshape(L, H, N),
                                     x[:, 2 * H * N:2 * H * N + H * P].reshape(L, H, P), (oracle.sigmoid(z) ** (1 / spec.tau)).reshape(L, H, N))
        gt = x[:, 2 * H * N + H * P:2 * H * N + 2 * H * P]
        want.append(D64((oracle.rms(o, 1e-5) * wn["norm"]).reshape(L, H * P) * gt * oracle.sigmoid(gt)))
    op = lambda u, meta, run: seqmix.gated_linear_attention(u, mod.a2, mod.a2_b, mod.norm_w, run.ssm, meta, H, N, P, spec.tau, 1e-5)
    for cuts in ((600,), (100, 20, 1), (7,)):
        got, _ = run_mixer(op, _Spec(gla=spec), us, cuts, "cuda", torch.bfloat16)
        for a, b in zip(got, want):
            assert (a.double() - b).abs().max().item() < 2e-2 * max(1.0, b.abs().max().item()), cuts


@pytest.mark.gpu
@pytest.mark.parametrize("H,D,R,Dv,kr", [(6, 32, 32, 48, 96), (16, 64, 32, 64, 128), (3, 64, 64, 32, 128), (4, 128, 64, 128, 256), (5, 24, 8, 40, 40)])
def test_bf16_latent_attention_over_long_prompts(H, D, R, Dv, kr):
    """The matrix-core prompt kernel over latent rows (and the general kernel at 48-wide rows), the batched head
    expansions with their gate, and decode-sized steps with the expansions in the kernels, against float64."""
    from edgellm.models.mixers import LatentAttention
    W = 64
    g = torch.Generator().manual_seed(D + H)
    lin = lambda o, i: BF(torch.randn(o, i, generator=g) * i ** -0.5)
    m = latent(H, D, R, Dv, 48, kr, base=10000.0)["mixer"]
    w = {"dq": lin(48, W), "dq.norm": torch.ones(48), "uq": lin(H * (D + R), 48), "dkv": lin(kr + R, W), "dkv.norm": torch.ones(kr), "uk": lin(H * D, kr),
         "uv": lin(H * Dv, kr), "g": lin(H * Dv, W), "o": lin(W, H * Dv)}
    spec = LatentAttnSpec(heads=H, dim=D, rot_dim=R, vdim=Dv, q_rank=48, kv_rank=kr, scale=m["scale"], rot_dims=R, rot_base=10000.0, gate=True)
    mod = LatentAttention(spec, W, 1e-5, torch.bfloat16, torch.device("cuda"))
    mod.proj_in.weight.copy_(torch.cat([w["dq"], w["dkv"], w["g"]])), mod.q_norm.copy_(w["dq.norm"]), mod.kv_norm.copy_(w["dkv.norm"])
    mod.uq.weight.copy_(w["uq"]), mod.o.weight.copy_(w["o"])
    mod.uk.copy_(w["uk"].view(H, D, kr)), mod.uv.copy_(w["uv"].view(H, Dv, kr).transpose(1, 2))
    hs = [BF(torch.randn(L, W, generator=g)) for L in (150, 65)]
    want = [D64(oracle.latent_attention(h.double().numpy(), {k: v.double().numpy() for k, v in w.items()}, "", m, 1e-5)) for h in hs]
    for cuts in ((150,), (60, 1, 30), (5,)):
        got, _ = run_mixer(mod, _Spec(latent=spec), hs, cuts, "cuda", torch.bfloat16)
        for a, b in zip(got, want):
            assert (a.double() - b).abs().max().item() < 4e-2 * max(1.0, b.abs().max().item()), cuts


@pytest.mark.gpu
@pytest.mark.parametrize("precision", ["fp32", "bf16"])
def test_sizes_that_are_not_multiples_of_eight(tmp_path, precision):
    """Odd widths and head sizes take the scalar kernel paths and unaligned slices of the fused projections."""
    cfg = CONFIGS["plain"]()
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
