"""Prefill / decode throughput of a layer-spec model beside the closest existing model of equal size
(``bench.py --hybrid-compare``): the Nudadra hybrid beside the parallel-residual row-cache decoder,
or (``--hybrid-family pagonex``) the Pagonex model (latent attention and gated delta-rule layers,
mixture-of-experts feed-forwards) beside the Nudadra hybrid, its closest relative: the same engine,
windowed attention over the paged cache, a recurrent mixer and a feed-forward per layer; or
(``--hybrid-family vetevik``) the Vetevik model (chunked attention whose values are its keys, a gated
delta rule with per-head decays, sigmoid-routed experts, norms on both sides of every sublayer)
beside the Pagonex model of equal width, heads, state size and active expert width; or
(``--hybrid-family fikupel``) the Fikupel model (latent attention without positions and gated
grouped-query attention with rotated values, both with a window and a sink, PolyNorm and expert
feed-forwards, two residual streams) beside the Vetevik model of equal width, heads, head size, window
and active expert width; or (``--hybrid-family numizen``) the Numizen model (gated latent attention and
gated linear attention beside a gelu-gated unit or group-limited squared-ReLU experts) beside the Pagonex
model of equal width, heads, head sizes, latent ranks, state size and active feed-forward work, its latent
attention without a window as well; or (``--hybrid-family felavik``) the Felavik model (gated attention with a
distance bias side by side with retention, lightning attention, group-limited silu-gated experts) beside the
Numizen model (the like recurrence and router) and the Fikupel model without window or kept tokens and with
one residual stream (the like attention and layer form), both of equal width, heads, head and state sizes and
active expert width.

Sizes resemble real layers (random weights): the hybrid layer has windowed attention with pooled
blocks + a Mamba-2 mixer + a squared-ReLU feed-forward; the comparison model is the
parallel-residual decoder (Phi layout: one norm, attention and MLP side by side) with the same
width, layer count, attention heads, head size, feed-forward width and vocabulary, bf16.

Per size: prefill tokens/s of one prompt of ``prompt`` tokens, decode tokens/s and ms/step of
``batch`` sequences at that context, and per-op times of one prefill and one decode step of the
hybrid (device events around each ``ops.seqmix`` call) with the bytes / flops each moves, so an op
can be priced against the 8 TB/s / 2.5 PFLOP/s roofline.
"""
from __future__ import annotations

import time
from typing import Dict, List

import torch

from ..models.configs import (ChunkAttnSpec, DecayAttnSpec, DeltaSpec, GatedAttnSpec, GLASpec, LatentAttnSpec, LayerSpec, ModelConfig, MoESpec,
                              SSDSpec, WindowAttnSpec, PRESETS)
from ..models.decoder import build_model
from ..models.hybrid import build_hybrid
from .generate import Generator, SamplingParams
from .ragged import RaggedEngine

SIZES = {
    "w1024": dict(width=1024, layers=4, heads=16, kv=4, dim=64, window=512, pool=16, s_heads=16, s_vdim=64, state=64,
                  ff=4096, vocab=32000),
    "w2048": dict(width=2048, layers=4, heads=16, kv=4, dim=128, window=1024, pool=32, s_heads=32, s_vdim=64,
                  state=128, ff=8192, vocab=32000),
    "w4096": dict(width=4096, layers=2, heads=32, kv=8, dim=128, window=2048, pool=64, s_heads=64, s_vdim=64,
                  state=128, ff=14336, vocab=32000),
}


def hybrid_config(s: dict) -> ModelConfig:
    a = WindowAttnSpec(s["heads"], s["kv"], s["dim"], s["dim"], s["dim"] ** -0.5, s["window"], s["pool"], s["dim"],
                       500000.0, {"rope_type": "yarn", "factor": 4.0, "original": 4096, "fast": 32.0, "slow": 1.0})
    m = SSDSpec(s["s_heads"], s["s_vdim"], s["state"], 1, 4, 1)
    specs = [LayerSpec("parallel", a, m, s["ff"]) for _ in range(s["layers"])]
    return ModelConfig(arch="nudadra", vocab_size=s["vocab"], hidden_size=s["width"], num_layers=s["layers"],
                       num_heads=s["heads"], num_kv_heads=s["kv"], intermediate_size=s["ff"], head_dim=s["dim"],
                       max_position_embeddings=1 << 20, norm="rms_scalar", norm_eps=1e-6, act="relu2",
                       parallel_residual=True, shared_input_norm=True, name="nudadra-bench", layer_specs=specs,
                       embed_scale=1.0)


# Pagonex sizes: per layer pair one latent-attention layer (the second reads the first one's cache) and one
# delta-rule layer; the experts' active width (top x ff + shared) equals the dense feed-forward of the
# Nudadra size of the same name
PAGONEX_SIZES = {
    "w1024": dict(width=1024, layers=4, heads=16, dim=64, rot=32, vdim=64, q_rank=384, kv_rank=128, window=512,
                  d_heads=16, d_dim=64, d_vdim=64, experts=16, top=3, ff=1024, shared=1024, vocab=32000),
    "w2048": dict(width=2048, layers=4, heads=16, dim=128, rot=64, vdim=128, q_rank=768, kv_rank=256, window=1024,
                  d_heads=16, d_dim=128, d_vdim=128, experts=32, top=3, ff=2048, shared=2048, vocab=32000),
}


def pagonex_config(s: dict) -> ModelConfig:
    yarn = {"rope_type": "yarn", "factor": 4.0, "original": 4096, "fast": 32.0, "slow": 1.0}
    moe = MoESpec(s["experts"], s["top"], 2.0, s["ff"], 7.0, s["shared"], 7.0)
    specs = []
    for i in range(s["layers"]):
        if i % 2 == 0:
            a = LatentAttnSpec(s["heads"], s["dim"], s["rot"], s["vdim"], s["q_rank"], s["kv_rank"],
                               (s["dim"] + s["rot"]) ** -0.5, s["window"], s["rot"], 500000.0, yarn,
                               kv_from=0 if i else None)
            specs.append(LayerSpec("latent_attention", latent=a, moe=moe))
        else:
            d = DeltaSpec(s["d_heads"], s["d_heads"], s["d_dim"], s["d_vdim"], 4, max(16, s["width"] // 32),
                          max(16, s["width"] // 32))
            specs.append(LayerSpec("channel_delta", delta=d, moe=moe))
    return ModelConfig(arch="pagonex", vocab_size=s["vocab"], hidden_size=s["width"], num_layers=s["layers"],
                       num_heads=s["heads"], num_kv_heads=1, intermediate_size=0, head_dim=1,
                       max_position_embeddings=1 << 20, norm="layer", norm_eps=1e-6, act="glu_clamp", name="pagonex-bench",
                       layer_specs=specs, canon_taps=4, bigram={"buckets": 8191, "mul_prev": 131, "mul_cur": 17},
                       logit_scale=1.0)


# Vetevik sizes: attention and delta-rule layers alternate as in the Pagonex size of the same name, with its
# width, head count, head sizes, state size and expert width; four experts per token make the active
# feed-forward width equal to Pagonex's three + shared; the chunk is as long as Pagonex's window
VETEVIK_SIZES = {
    "w1024": dict(width=1024, layers=4, heads=16, kv=4, dim=64, chunk=512, softcap=50.0, d_heads=16, d_dim=64, d_vdim=64,
                  experts=16, top=4, ff=1024, groups=2, vocab=32000),
    "w2048": dict(width=2048, layers=4, heads=16, kv=4, dim=128, chunk=1024, softcap=50.0, d_heads=16, d_dim=128,
                  d_vdim=128, experts=32, top=4, ff=2048, groups=2, vocab=32000),
}


def vetevik_config(s: dict) -> ModelConfig:
    moe = MoESpec(s["experts"], s["top"], 1.0, s["ff"], router="sigmoid", act="silu_glu", weight_on="input")
    specs = []
    for i in range(s["layers"]):
        if i % 2 == 0:
            a = ChunkAttnSpec(s["heads"], s["kv"], s["dim"], s["dim"] ** -0.5, s["chunk"], s["softcap"])
            specs.append(LayerSpec("chunk_attention", chunk_attn=a, moe=moe))
        else:
            d = DeltaSpec(s["d_heads"], s["d_heads"], s["d_dim"], s["d_vdim"], 4, decay="head")
            specs.append(LayerSpec("head_delta", delta=d, moe=moe))
    return ModelConfig(arch="vetevik", vocab_size=s["vocab"], hidden_size=s["width"], num_layers=s["layers"],
                       num_heads=s["heads"], num_kv_heads=s["kv"], intermediate_size=0, head_dim=s["dim"],
                       max_position_embeddings=1 << 20, norm="rms_group", norm_eps=1e-6, act="silu_glu", pos_emb="none",
                       tie_word_embeddings=True, name="vetevik-bench", layer_specs=specs, norm_groups=s["groups"],
                       residual_mult=0.3)


# Fikupel sizes: latent-attention and gated-attention layers alternate; width, head count, head sizes, window
# (= Vetevik's chunk) and experts as in the Vetevik size of the same name, latent ranks as in the Pagonex one;
# the first layer's PolyNorm feed-forward is as wide as the experts' active width
FIKUPEL_SIZES = {
    "w1024": dict(width=1024, layers=4, heads=16, kv=4, dim=64, window=512, keep=4, rot=32, q_rank=384, kv_rank=128,
                  experts=16, top=4, ff=1024, dense_ff=4096, streams=2, vocab=32000),
    "w2048": dict(width=2048, layers=4, heads=16, kv=4, dim=128, window=1024, keep=4, rot=64, q_rank=768, kv_rank=256,
                  experts=32, top=4, ff=2048, dense_ff=8192, streams=2, vocab=32000),
}


def fikupel_config(s: dict) -> ModelConfig:
    """``window`` None and ``keep`` 0: every earlier token is seen; ``streams`` 1: the plain residual sum."""
    moe = MoESpec(s["experts"], s["top"], 1.0, s["ff"], router="top_softmax", act="silu_glu", weight_on="output",
                  router_bias=True)
    llama3 = {"rope_type": "llama3", "factor": 8.0, "low_freq_factor": 1.0, "high_freq_factor": 4.0,
              "original_max_position_embeddings": 8192.0}
    specs = []
    for i in range(s["layers"]):
        ff = dict(ff=s["dense_ff"], ff_act="polynorm") if i == 0 else dict(moe=moe, ff_act="polynorm")
        if i % 2 == 0:
            a = LatentAttnSpec(s["heads"], s["dim"], 0, s["dim"], s["q_rank"], s["kv_rank"], s["dim"] ** -0.5, s["window"],
                               sink=True)
            specs.append(LayerSpec("latent_attention", latent=a, **ff))
        else:
            a = GatedAttnSpec(s["heads"], s["kv"], s["dim"], s["dim"], s["dim"] ** -0.5, s["window"], s["keep"], s["rot"],
                              500000.0, llama3)
            specs.append(LayerSpec("gated_attention", gated_attn=a, **ff))
    return ModelConfig(arch="fikupel", vocab_size=s["vocab"], hidden_size=s["width"], num_layers=s["layers"],
                       num_heads=s["heads"], num_kv_heads=s["kv"], intermediate_size=0, head_dim=s["dim"],
                       max_position_embeddings=1 << 20, norm="rms", norm_eps=1e-6, act="silu_glu", pos_emb="rope",
                       tie_word_embeddings=True, name="fikupel-bench", layer_specs=specs, streams=s["streams"],
                       hyper=s["streams"] > 1)


# Numizen sizes: latent-attention and linear-attention layers alternate with the heads, ranks and state sizes of the
# Pagonex size of the same name; a squared-ReLU expert has two matrices where Pagonex's gated one has three, so
# experts half as wide again make the active work equal; the first layer's dense unit is as wide as Pagonex's
# three experts + shared one
NUMIZEN_SIZES = {
    "w1024": dict(width=1024, layers=4, heads=16, dim=64, rot=32, vdim=64, q_rank=384, kv_rank=128, l_heads=16, l_dim=64,
                  l_vdim=64, rank=16, experts=16, top=3, groups=4, keep=2, ff=1536, shared=1536, dense_ff=4096, vocab=32000),
    "w2048": dict(width=2048, layers=4, heads=16, dim=128, rot=64, vdim=128, q_rank=768, kv_rank=256, l_heads=16, l_dim=128,
                  l_vdim=128, rank=16, experts=32, top=3, groups=4, keep=2, ff=3072, shared=3072, dense_ff=8192, vocab=32000),
}


def numizen_config(s: dict) -> ModelConfig:
    moe = MoESpec(s["experts"], s["top"], 1.0, s["ff"], shared_ff=s["shared"], router="softmax", act="relu2", correction=True,
                  groups=s["groups"], groups_keep=s["keep"], shared_gate=True)
    specs = []
    for i in range(s["layers"]):
        ff = dict(ff=s["dense_ff"], ff_act="gelu_glu") if i == 0 else dict(moe=moe, ff_act="gelu_glu")
        if i % 2 == 0:
            a = LatentAttnSpec(s["heads"], s["dim"], s["rot"], s["vdim"], s["q_rank"], s["kv_rank"], (s["dim"] + s["rot"]) ** -0.5,
                               None, s["rot"], 500000.0, gate=True)
            specs.append(LayerSpec("latent_attention", latent=a, **ff))
        else:
            specs.append(LayerSpec("gla", gla=GLASpec(s["l_heads"], s["l_dim"], s["l_vdim"], 16.0, s["rank"]), **ff))
    return ModelConfig(arch="numizen", vocab_size=s["vocab"], hidden_size=s["width"], num_layers=s["layers"],
                       num_heads=s["heads"], num_kv_heads=1, intermediate_size=s["dense_ff"], head_dim=s["dim"],
                       max_position_embeddings=1 << 15, norm="dyt", norm_eps=1e-6, act="gelu_tanh", parallel_residual=True,
                       pos_emb="learned", name="numizen-bench", layer_specs=specs, layer_scale=True)


# Felavik sizes: parallel (attention beside retention) and lightning layers alternate; heads, head sizes, state sizes and
# experts as in the Fikupel / Numizen sizes of the same name, the active expert width as in Fikupel
FELAVIK_SIZES = {
    "w1024": dict(width=1024, layers=4, heads=16, kv=4, dim=64, vdim=64, buckets=32, far=512, r_heads=16, r_dim=64, r_vdim=64,
                  experts=16, top=4, groups=4, keep=2, ff=1024, vocab=32000),
    "w2048": dict(width=2048, layers=4, heads=16, kv=4, dim=128, vdim=128, buckets=32, far=1024, r_heads=16, r_dim=128,
                  r_vdim=128, experts=32, top=4, groups=4, keep=2, ff=2048, vocab=32000),
}


def felavik_config(s: dict) -> ModelConfig:
    moe = MoESpec(s["experts"], s["top"], 1.0, s["ff"], act="silu_glu", groups=s["groups"], groups_keep=s["keep"])
    decay = tuple(1.0 - 2.0 ** (-2.0 - 8.0 * h / s["r_heads"]) for h in range(s["r_heads"]))
    specs = []
    for i in range(s["layers"]):
        if i % 2 == 0:
            a = GatedAttnSpec(s["heads"], s["kv"], s["dim"], s["vdim"], s["dim"] ** -0.5, rotate_values=False, temp=False, sink=False,
                              qkv_bias=True, q_temp=(0.3, 1024), rel_buckets=s["buckets"], rel_max=s["far"])
            r = DecayAttnSpec(s["r_heads"], s["r_dim"], s["r_vdim"], decay, rot_dims=s["r_dim"], rot_base=500000.0,
                              k_scale=s["r_dim"] ** -0.5)
            specs.append(LayerSpec("attention_retention", moe=moe, gated_attn=a, decay_attn=r, left_scale=0.7, right_scale=0.7))
        else:
            d = DecayAttnSpec(s["r_heads"], s["r_dim"], s["r_vdim"], decay, act="silu", norm="all", gate_act="sigmoid")
            specs.append(LayerSpec("lightning", moe=moe, decay_attn=d))
    return ModelConfig(arch="felavik", vocab_size=s["vocab"], hidden_size=s["width"], num_layers=s["layers"],
                       num_heads=s["heads"], num_kv_heads=s["kv"], intermediate_size=0, head_dim=s["dim"],
                       max_position_embeddings=1 << 20, norm="rms", norm_eps=1e-6, act="silu_glu", pos_emb="rope",
                       name="felavik-bench", layer_specs=specs, streams=1, hyper=False, logit_softcap=30.0)


def closest_config(s: dict) -> ModelConfig:
    return PRESETS["phi-2"].replace(vocab_size=s["vocab"], hidden_size=s["width"], num_layers=s["layers"],
                                    num_heads=s["heads"], num_kv_heads=s["kv"], head_dim=s["dim"], rotary_dim=s["dim"],
                                    intermediate_size=s["ff"], max_position_embeddings=1 << 16, name="phi-layout")


def _timed(fn, reps: int, warm: int = 1) -> float:
    for _ in range(warm):
        fn()
    torch.cuda.synchronize()
    t0 = time.perf_counter()
    for _ in range(reps):
        fn()
    torch.cuda.synchronize()
    return (time.perf_counter() - t0) / reps


def bench_hybrid(s: dict, prompt: int, batch: int, steps: int, device, cfg: ModelConfig = None) -> Dict:
    model = build_hybrid(cfg if cfg is not None else hybrid_config(s), torch.bfloat16, device, seed=0)
    ids = torch.randint(0, s["vocab"], (prompt,), generator=torch.Generator().manual_seed(0)).tolist()
    page = 64
    eng = RaggedEngine(model, (batch + 1) * ((prompt + steps + 2 * page) // page) * page, slots=batch + 1)

    def prefill():
        eng.step([("p", ids, [prompt - 1])])
        eng.close("p")
    t_pre = _timed(prefill, 3)
    for b in range(batch):
        eng.step([(b, ids, [prompt - 1])])
    tok = [1] * batch
    dec = lambda: eng.step([(b, [tok[b]], [0]) for b in range(batch)])
    t_dec = _timed(dec, steps, warm=3)
    out = {"prefill_tok_s": prompt / t_pre, "prefill_ms": t_pre * 1e3, "decode_tok_s": batch / t_dec,
           "decode_ms_per_step": t_dec * 1e3, "decode_graph": bool(getattr(eng, "graphs_used", False)),
           "ops_prefill_us": op_times(eng, [("q", ids, [prompt - 1])], close=["q"]),
           "ops_decode_us": op_times(eng, [(b, [tok[b]], [0]) for b in range(batch)])}
    return out


def op_times(eng: RaggedEngine, entries, close=()) -> Dict[str, float]:
    """Device time per op kind over one step (sum over layers), from events around every
    ``ops.seqmix`` call and every projection (eager step: no graph)."""
    from ..ops import seqmix
    import torch.nn.functional as F
    marks: List[tuple] = []
    names = ["embedding_scaled", "scalar_rms_norm", "relu2", "cat_cast", "combine_residual", "gated_group_norm",
             "rope_paged_write", "pool_blocks", "window_pool_attention", "conv_silu", "ssd_scan", "linear_f32",
             "embedding_bigram", "canon_conv", "layer_norm_rows", "layer_norm_residual", "rms_norm_cols", "glu_clamp",
             "latent_write", "delta_prepare", "delta_rule_scan", "head_norm_gate", "moe_route", "moe_experts",
             "group_rms_norm", "group_norm_residual", "chunk_attention", "delta_prepare_head", "glu_silu",
             "hyper_read_norm", "hyper_update", "poly_norm", "qk_norm_rope_write", "unrotate_gate",
             "embedding_learned", "parallel_update", "glu_gelu", "moe_route_grouped", "moe_experts_shared",
             "latent_expand_write", "head_expand_gate", "gated_linear_attention", "decay_linear_attention", "softcap"]
    saved = {n: getattr(seqmix, n) for n in names}
    lin = F.linear

    depth = [0]                                  # an op inside another op counts for the outer one

    def wrap(name, fn):
        def inner(*a, **k):
            if depth[0]:
                return fn(*a, **k)
            depth[0] += 1
            e0, e1 = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
            e0.record()
            try:
                r = fn(*a, **k)
            finally:
                depth[0] -= 1
            e1.record()
            marks.append((name, e0, e1))
            return r
        return inner
    graphs = getattr(eng, "use_graphs", None)
    try:
        if graphs is not None:
            eng.use_graphs = False
        for n in names:
            setattr(seqmix, n, wrap(n, saved[n]))
        from ..models import layers as L
        orig_fwd = L.Linear.forward
        L.Linear.forward = wrap("projections", orig_fwd)
        bmm = torch.bmm
        torch.bmm = wrap("head_expansions_bmm", bmm)
        eng.step(entries)
        torch.cuda.synchronize()
    finally:
        for n in names:
            setattr(seqmix, n, saved[n])
        L.Linear.forward = orig_fwd
        torch.bmm = bmm
        if graphs is not None:
            eng.use_graphs = graphs
    for r in close:
        eng.close(r)
    out: Dict[str, float] = {}
    for name, e0, e1 in marks:
        out[name] = out.get(name, 0.0) + e0.elapsed_time(e1) * 1e3
    return {k: round(v, 1) for k, v in out.items()}


def bench_closest(s: dict, prompt: int, batch: int, steps: int, device) -> Dict:
    cfg = closest_config(s)
    model = build_model(cfg, torch.bfloat16, device, seed=0)
    gen = Generator(model, max_batch=batch, max_seq=prompt + steps + 16)
    gen.b1 = False
    ids = torch.randint(0, s["vocab"], (1, prompt), generator=torch.Generator().manual_seed(0)).to(device)
    t_pre = _timed(lambda: gen.prefill(ids, 0, 0), 3)
    sp = SamplingParams(max_new_tokens=steps + 8, do_sample=False, repetition_penalty=1.0)
    gen.start([ids[0].tolist()] * batch, sp)
    gen.step(3, record_latency=False)
    torch.cuda.synchronize()
    t0 = time.perf_counter()
    gen.step(steps, record_latency=False)
    torch.cuda.synchronize()
    t_dec = (time.perf_counter() - t0) / steps
    return {"prefill_tok_s": prompt / t_pre, "prefill_ms": t_pre * 1e3, "decode_tok_s": batch / t_dec,
            "decode_ms_per_step": t_dec * 1e3}


def run_pagonex(sizes: List[str], prompt: int, batch: int, steps: int, device) -> Dict:
    res = {}
    r2 = lambda d: {k: (round(v, 2) if isinstance(v, float) else v) for k, v in d.items()}
    for name in sizes:
        s = PAGONEX_SIZES[name]
        p = bench_hybrid(s, prompt, batch, steps, device, pagonex_config(s))
        torch.cuda.empty_cache()
        h = bench_hybrid(SIZES[name], prompt, batch, steps, device)
        torch.cuda.empty_cache()
        res[name] = {"size": s, "closest_size": SIZES[name], "pagonex": r2(p), "closest_nudadra": r2(h),
                     "prefill_ratio": round(p["prefill_tok_s"] / h["prefill_tok_s"], 3),
                     "decode_ratio": round(p["decode_tok_s"] / h["decode_tok_s"], 3)}
    return {"metric": "prefill / decode tokens/s, Pagonex layer-spec model vs the Nudadra hybrid of equal size",
            "dtype": "bf16", "data": "synthetic (random weights, random prompt)", "prompt_tokens": prompt,
            "decode_batch": batch, "decode_steps": steps, "sizes": res}


def run_vetevik(sizes: List[str], prompt: int, batch: int, steps: int, device) -> Dict:
    res = {}
    r2 = lambda d: {k: (round(v, 2) if isinstance(v, float) else v) for k, v in d.items()}
    for name in sizes:
        s, c = VETEVIK_SIZES[name], PAGONEX_SIZES[name]
        v = bench_hybrid(s, prompt, batch, steps, device, vetevik_config(s))
        torch.cuda.empty_cache()
        p = bench_hybrid(c, prompt, batch, steps, device, pagonex_config(c))
        torch.cuda.empty_cache()
        res[name] = {"size": s, "closest_size": c, "vetevik": r2(v), "closest_pagonex": r2(p),
                     "prefill_ratio": round(v["prefill_tok_s"] / p["prefill_tok_s"], 3),
                     "decode_ratio": round(v["decode_tok_s"] / p["decode_tok_s"], 3)}
    return {"metric": "prefill / decode tokens/s, Vetevik layer-spec model vs the Pagonex model of equal size",
            "dtype": "bf16", "data": "synthetic (random weights, random prompt)", "prompt_tokens": prompt,
            "decode_batch": batch, "decode_steps": steps, "sizes": res}


def run_fikupel(sizes: List[str], prompt: int, batch: int, steps: int, device) -> Dict:
    res = {}
    r2 = lambda d: {k: (round(v, 2) if isinstance(v, float) else v) for k, v in d.items()}
    for name in sizes:
        s, c = FIKUPEL_SIZES[name], VETEVIK_SIZES[name]
        f = bench_hybrid(s, prompt, batch, steps, device, fikupel_config(s))
        torch.cuda.empty_cache()
        v = bench_hybrid(c, prompt, batch, steps, device, vetevik_config(c))
        torch.cuda.empty_cache()
        res[name] = {"size": s, "closest_size": c, "fikupel": r2(f), "closest_vetevik": r2(v),
                     "prefill_ratio": round(f["prefill_tok_s"] / v["prefill_tok_s"], 3),
                     "decode_ratio": round(f["decode_tok_s"] / v["decode_tok_s"], 3)}
    return {"metric": "prefill / decode tokens/s, Fikupel layer-spec model vs the Vetevik model of equal size",
            "dtype": "bf16", "data": "synthetic (random weights, random prompt)", "prompt_tokens": prompt,
            "decode_batch": batch, "decode_steps": steps, "sizes": res}


def run_numizen(sizes: List[str], prompt: int, batch: int, steps: int, device) -> Dict:
    res = {}
    r2 = lambda d: {k: (round(v, 2) if isinstance(v, float) else v) for k, v in d.items()}
    for name in sizes:
        s, c = NUMIZEN_SIZES[name], dict(PAGONEX_SIZES[name], window=None)
        n = bench_hybrid(s, prompt, batch, steps, device, numizen_config(s))
        torch.cuda.empty_cache()
        p = bench_hybrid(c, prompt, batch, steps, device, pagonex_config(c))
        torch.cuda.empty_cache()
        res[name] = {"size": s, "closest_size": c, "numizen": r2(n), "closest_pagonex": r2(p),
                     "prefill_ratio": round(n["prefill_tok_s"] / p["prefill_tok_s"], 3),
                     "decode_ratio": round(n["decode_tok_s"] / p["decode_tok_s"], 3)}
    return {"metric": "prefill / decode tokens/s, Numizen layer-spec model vs the Pagonex model of equal size",
            "dtype": "bf16", "data": "synthetic (random weights, random prompt)", "prompt_tokens": prompt,
            "decode_batch": batch, "decode_steps": steps, "sizes": res}


def run_felavik(sizes: List[str], prompt: int, batch: int, steps: int, device) -> Dict:
    res = {}
    r2 = lambda d: {k: (round(v, 2) if isinstance(v, float) else v) for k, v in d.items()}
    for name in sizes:
        s, n, f = FELAVIK_SIZES[name], NUMIZEN_SIZES[name], dict(FIKUPEL_SIZES[name], window=None, keep=0, streams=1)
        got = {}
        for label, cfg, size in (("felavik", felavik_config(s), s), ("closest_numizen", numizen_config(n), n),
                                 ("closest_fikupel", fikupel_config(f), f)):
            got[label] = bench_hybrid(size, prompt, batch, steps, device, cfg)
            torch.cuda.empty_cache()
        res[name] = {"size": s, "closest_size": n, "closest_attention_size": f, **{k: r2(v) for k, v in got.items()}}
        for k in ("numizen", "fikupel"):
            for what in ("prefill", "decode"):
                res[name][f"{what}_ratio_{k}"] = round(got["felavik"][f"{what}_tok_s"] / got[f"closest_{k}"][f"{what}_tok_s"], 3)
    return {"metric": "prefill / decode tokens/s, Felavik layer-spec model vs the Numizen and Fikupel models of equal size",
            "dtype": "bf16", "data": "synthetic (random weights, random prompt)", "prompt_tokens": prompt,
            "decode_batch": batch, "decode_steps": steps, "sizes": res}


def run(sizes: List[str], prompt: int = 4096, batch: int = 4, steps: int = 32, device=None, family: str = "nudadra") -> Dict:
    device = torch.device(device or "cuda:0")
    if family == "pagonex":
        return run_pagonex(sizes, prompt, batch, steps, device)
    if family == "vetevik":
        return run_vetevik(sizes, prompt, batch, steps, device)
    if family == "fikupel":
        return run_fikupel(sizes, prompt, batch, steps, device)
    if family == "numizen":
        return run_numizen(sizes, prompt, batch, steps, device)
    if family == "felavik":
        return run_felavik(sizes, prompt, batch, steps, device)
    res = {}
    for name in sizes:
        s = SIZES[name]
        h = bench_hybrid(s, prompt, batch, steps, device)
        torch.cuda.empty_cache()
        c = bench_closest(s, prompt, batch, steps, device)
        torch.cuda.empty_cache()
        r2 = lambda d: {k: (round(v, 2) if isinstance(v, float) else v) for k, v in d.items()}
        res[name] = {"size": s, "nudadra": r2(h), "closest_phi_layout": r2(c),
                     "prefill_ratio": round(h["prefill_tok_s"] / c["prefill_tok_s"], 3),
                     "decode_ratio": round(h["decode_tok_s"] / c["decode_tok_s"], 3)}
    return {"metric": "prefill / decode tokens/s, Nudadra layer-spec model vs the parallel-residual decoder of equal size",
            "dtype": "bf16", "data": "synthetic (random weights, random prompt)", "prompt_tokens": prompt,
            "decode_batch": batch, "decode_steps": steps, "sizes": res}
