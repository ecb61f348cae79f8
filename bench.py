#!/usr/bin/env python3
"""Decode and prefill throughput of the engine at Qwen3-8B layer sizes on one MI355X.

    python bench.py [--gpus 1] [--steps K] [--warmup W]

Prints ONE JSON line.  `value` is decoded tokens per second at batch 8 and the context
length the configuration names (the last timed step ends at that length); a "step" is one
decode step through the engine's own step function (mixed-batch path, paged cache,
kernels) followed by greedy sampling on the GPU, launched as the engine launches its steps:
the sampled ids reach the next step on the device and travel to the host beside it, so the
host prepares a step while the GPU runs the one before (the timed steps lie between two
synchronizations, and all of their tokens have reached the host at the second).  Beside it: the prefill of one
2,048-token prompt, the decode step's bandwidth roofline, decode at batch 1 and 64 (`points`,
and each one's own roofline in `points_roofline`), and decode at batch 8 with four times the
context (`further`).

`--product M,N,K[,slices[,shape]]` times one bfloat16 product alone, in the hand-written many-row
tiled kernel and in the vendor library.

`--peaks` adds what this card itself reaches (a read-only stream, one large square product) and
the fractions of those, beside the fractions of the published peaks that the line always has.

Data is synthetic: weights are seeded random values of the architecture's shapes made
on the GPU, token ids are seeded uniform, and the cache contents the decode steps read
are random values (decode timing does not depend on what the cache holds).

`--workload serve14b` and `--workload long32b` instead run the two serving workloads of the
larger configurations through the whole engine (scheduler, chunked prefill, continuous
batching, greedy sampling) and print their own JSON line: total generated tokens per second.
`--workload many06b` is the one run the reference publishes a figure for (Qwen3-0.6B, 256
concurrent requests, 1,024 new tokens each); its line carries the ratio to that figure, which
was measured on other hardware.  `--workload many8b` is 192 concurrent requests (prompts of 64
to 512 tokens, 256 new tokens each) at Qwen3-8B sizes: decode steps of 129 to 256 rows.

`--design mufenex[:SIZE]` times the Mufenex family (windowed attention with a soft cap and a distance
bias, sublayer outputs normed, dense gelu or routed silu feed-forwards) beside Qwen3 at equal sizes
(the same width, heads, head size, feed-forward width, window, vocabulary and number of layers): the
prefill of one prompt and a decode step at batch 8, one JSON line with both.
`--design lilalorn[:SIZE]` times the Lilalorn family (layers of softmax attention beside retention, and of
gated linear attention, in turn; experts without a gate and a shared one) beside the closest family there
is, Mufenex with routed experts and no window, at equal sizes.
`--design debusun[:SIZE]` times the Debusun family (layers of attention over a latent with sinks and a gate, of
windowed attention whose heads are normed after the rotation, and of a selective state space, in turn; dense
feed-forwards of a squared relu; a table of token pairs beside the embedding) beside dense Mufenex at equal sizes.
`--design vuzazen[:SIZE]` times the Vuzazen family (layers of attention over a latent with the queries through a latent
of their own, of a matrix memory, and of attention behind a short convolution whose heads' scores are mixed, in turn;
dense silu feed-forwards, or experts that see the token times its score) beside Debusun at equal sizes, which has no
experts: at the size with experts its feed-forwards are dense of the same active width.
`--design tisosun[:SIZE]` times the Tisosun family beside dense Mufenex, `--design litizen[:SIZE]` the Litizen family (layers
of windowed attention whose values are its keys, of a selective state space, of attention within chunks whose values turn, and
of the state space again; dense feed-forwards, or experts beside identity experts and a shared one) beside Debusun, whose
feed-forwards are dense at every size.
"""
from __future__ import annotations

import argparse
import json
import sys
import time

# MI355X published peaks
HBM_GBPS = 8000.0
PEAK_TFLOPS = {"bf16": 2500.0, "fp16": 2500.0, "fp8": 5000.0, "fp32": 157.3}

QWEN3_8B = dict(
    architectures=["Qwen3ForCausalLM"], hidden_size=4096, intermediate_size=12288,
    num_hidden_layers=36, num_attention_heads=32, num_key_value_heads=8, head_dim=128,
    vocab_size=151936, rope_theta=1e6, rms_norm_eps=1e-6, tie_word_embeddings=False,
    max_position_embeddings=40960, hidden_act="silu")
QWEN3_14B = dict(QWEN3_8B, hidden_size=5120, intermediate_size=17408, num_hidden_layers=40,
                 num_attention_heads=40, num_key_value_heads=8)
QWEN3_32B = dict(QWEN3_8B, hidden_size=5120, intermediate_size=25600, num_hidden_layers=64,
                 num_attention_heads=64, num_key_value_heads=8)
QWEN3_0_6B = dict(QWEN3_8B, hidden_size=1024, intermediate_size=3072, num_hidden_layers=28,
                  num_attention_heads=16, num_key_value_heads=8, tie_word_embeddings=True)
# the serving workloads of the two larger configurations, and the one the reference publishes a
# figure for: Qwen3-0.6B, 256 concurrent requests of 16 prompt tokens, 1,024 new tokens each
# (/root/reference/python/ReadMe.md:2-13: 10,944.62 generated tokens/s on a CUDA GPU)
WORKLOADS = {
    "many06b": dict(model=QWEN3_0_6B, name="Qwen3-0.6B layer sizes", requests=256, prompt=(16, 16), new_tokens=1024,
                    chunk=2048, max_model_len=1088, reference_tok_s=10944.62),
    "serve14b": dict(model=QWEN3_14B, name="Qwen3-14B layer sizes", requests=64, prompt=(128, 2048), new_tokens=256,
                     chunk=2048, max_model_len=2304),
    "many8b": dict(model=QWEN3_8B, name="Qwen3-8B layer sizes", requests=192, prompt=(64, 512), new_tokens=256,
                   chunk=2048, max_model_len=768),
    "long32b": dict(model=QWEN3_32B, name="Qwen3-32B layer sizes", requests=16, prompt=(8192, 8192), new_tokens=512,
                    chunk=2048, max_model_len=8704),
}
# sizes of the `--design` comparison: width, query heads, kv heads, head size, value head size, feed-forward width,
# window, experts (0: dense; else `experts` of `top`, each of ff / top so that a token's active width is ff)
DESIGN_SIZES = {
    "1k": dict(width=1024, heads=16, kv_heads=8, dim=128, vdim=128, ff=3072, window=1024, experts=0, top=0),
    "4k": dict(width=4096, heads=32, kv_heads=8, dim=128, vdim=128, ff=12288, window=2048, experts=0, top=0),
    "4k-moe": dict(width=4096, heads=32, kv_heads=8, dim=128, vdim=128, ff=12288, window=2048, experts=8, top=2),
    "2k-v": dict(width=2048, heads=16, kv_heads=4, dim=64, vdim=128, ff=8192, window=512, experts=16, top=2),
    "1k-moe": dict(width=1024, heads=16, kv_heads=8, dim=128, vdim=128, ff=3072, window=1024, experts=8, top=2),
    "2k-d": dict(width=2048, heads=16, kv_heads=4, dim=64, vdim=128, ff=8192, window=512, experts=0, top=0),
    # two kv heads: the heads' mix scores a query against both kv heads' dims at once (256 of them)
    "1k-g2": dict(width=1024, heads=16, kv_heads=2, dim=128, vdim=128, ff=3072, window=1024, experts=0, top=0),
    "4k-g2": dict(width=4096, heads=32, kv_heads=2, dim=128, vdim=128, ff=12288, window=2048, experts=0, top=0),
    "4k-g2-moe": dict(width=4096, heads=32, kv_heads=2, dim=128, vdim=128, ff=12288, window=2048, experts=8, top=2),
}
LILALORN_SIZES = ("1k-moe", "4k-moe", "2k-v")      # the sizes with experts: every Lilalorn layer has them
DEBUSUN_SIZES = ("1k", "4k")                        # the dense sizes: every Debusun feed-forward is dense
# Debusun's own sizes at every width: the latent and its turned part (together what the matrix-core kernel takes for
# one head), the state space's head and state sizes (its inner width is twice the model's)
DEBUSUN_LATENT = dict(kv_rank=192, rot_dim=64)
DEBUSUN_STATE = dict(vdim=64, state=128, groups=1, conv=4, norm_groups=1)
VUZAZEN_SIZES = ("1k-g2", "4k-g2", "4k-g2-moe")
# Vuzazen's own sizes at every width: the latents (keys as Debusun's; queries through 3/8 of the width), the memories'
# heads (a quarter as many as the query heads, keys as wide as the attention's and values twice that), the taps
VUZAZEN_LATENT = dict(kv_rank=192, rot_dim=64)
VUZAZEN_TAPS = 4
TISOSUN_SIZES = ("1k", "4k", "2k-d")
# Tisosun's own sizes at every width: recurrences as wide as the model (gates in as many blocks as there are query heads, 4
# taps), the linear attention's heads as Lilalorn's, half of a head turned, a token input of 256 columns a layer
TISOSUN_SIDE = 256
TISOSUN_TAPS = 4
LITIZEN_SIZES = ("1k", "4k", "4k-moe")
# Litizen's own sizes at every width: the state space as Debusun's, norms in 4 groups, 4 taps in front of every mixer, half of an
# attention_2 head turned; with experts, 2 identity experts beside them and a shared one as wide as an expert
LITIZEN_GROUPS, LITIZEN_TAPS, LITIZEN_IDENTITY = 4, 4, 2
DESIGN_CHOICES = {"mufenex": (tuple(k for k in DESIGN_SIZES if "g2" not in k and k != "2k-d"), "qwen3"), "lilalorn": (LILALORN_SIZES, "mufenex"),
                  "debusun": (DEBUSUN_SIZES, "mufenex"), "vuzazen": (VUZAZEN_SIZES, "debusun"),
                  "tisosun": (TISOSUN_SIZES, "mufenex"), "litizen": (LITIZEN_SIZES, "debusun")}
DESIGN_VOCAB = 32000
MODELS = {"0.6b": QWEN3_0_6B, "8b": QWEN3_8B, "14b": QWEN3_14B, "32b": QWEN3_32B}
CONTEXT = 4096
PREFILL_TOKENS = 2048


def weight_bytes(cfg, esize=2):
    h, i, nq, nkv, d, v, L = (cfg.hidden_size, cfg.intermediate_size, cfg.num_attention_heads,
                              cfg.num_key_value_heads, cfg.head_dim, cfg.vocab_size, cfg.num_hidden_layers)
    per_layer = (nq + 2 * nkv) * d * h + h * nq * d + 2 * i * h + h * i
    return (L * per_layer + v * h) * esize          # every linear weight once, and the head


def kv_bytes_per_token(cfg, esize=2):
    return 2 * cfg.num_key_value_heads * cfg.head_dim * esize * cfg.num_hidden_layers


def prefill_flops(cfg, T):
    h, i, nq, nkv, d, v, L = (cfg.hidden_size, cfg.intermediate_size, cfg.num_attention_heads,
                              cfg.num_key_value_heads, cfg.head_dim, cfg.vocab_size, cfg.num_hidden_layers)
    per_layer = (nq + 2 * nkv) * d * h + h * nq * d + 2 * i * h + h * i
    linear = 2.0 * T * L * per_layer + 2.0 * v * h          # the head runs on one row
    attn = L * 4.0 * nq * d * (T * (T + 1) / 2.0)           # causal QK^T and PV
    return linear + attn


def serve(workload: str, layers, run_ahead: bool = True) -> int:
    """One of the serving workloads through the whole engine."""
    import torch
    from xinfer_amd import EngineConfig, SamplingParams
    from xinfer_amd.engine import build_model
    from xinfer_amd.engine.llm_engine import LLMEngine
    from xinfer_amd.models import config_from_dict
    from xinfer_amd.weights.random_init import random_store_for

    w = WORKLOADS[workload]
    full = w["model"]["num_hidden_layers"]
    raw = dict(w["model"], num_hidden_layers=layers or full)
    _, cfg = config_from_dict(raw)
    t0 = time.time()
    model = build_model(cfg, random_store_for(cfg, seed=0), "bf16", "cuda:0")
    torch.cuda.synchronize()
    print(f"[bench] {w['name']}, {cfg.num_hidden_layers} layers, built in {time.time() - t0:.1f}s", file=sys.stderr, flush=True)
    page = 64
    n = w["requests"]
    pages = n * (-(-w["max_model_len"] // page)) + 8
    eng = LLMEngine(EngineConfig(max_num_seqs=n, max_model_len=w["max_model_len"], num_pages=pages, page_size=page,
                                 prefill_chunk_size=w["chunk"], seed=1, run_ahead=run_ahead),     # a step's token budget is the chunk
                    model=model)
    g = torch.Generator().manual_seed(4)
    lo, hi = w["prompt"]
    lens = [lo] * n if lo == hi else torch.randint(lo, hi + 1, (n,), generator=g).tolist()
    prompts = [torch.randint(0, cfg.vocab_size, (m,), generator=g).tolist() for m in lens]
    sp = SamplingParams(temperature=0.0, max_tokens=w["new_tokens"], ignore_eos=True)
    eng.generate(prompts[:2], SamplingParams(temperature=0.0, max_tokens=4, ignore_eos=True))   # warm-up
    steps0 = eng.steps
    eng.step_log = []
    torch.cuda.synchronize()
    t = time.perf_counter()
    outs = eng.generate(prompts, sp)
    torch.cuda.synchronize()
    dt = time.perf_counter() - t
    new = sum(o.decoded_length for o in outs)
    # The least time the steps that ran could take: a step reads every weight once and the cache of its
    # requests, and computes its tokens' products and its attention's pairs; it is bound by the slower
    # of the two at the published peaks.
    h, i_, nq, nkv, d, L = (cfg.hidden_size, cfg.intermediate_size, cfg.num_attention_heads, cfg.num_key_value_heads,
                            cfg.head_dim, cfg.num_hidden_layers)
    per_layer = (nq + 2 * nkv) * d * h + h * nq * d + 3 * i_ * h
    wb, kvb = weight_bytes(cfg), kv_bytes_per_token(cfg)
    least = mem_s = 0.0
    for tokens, keys, pairs in eng.step_log:
        mem = (wb + keys * kvb) / (HBM_GBPS * 1e9)
        flop = (2.0 * tokens * L * per_layer + L * 4.0 * nq * d * pairs) / (PEAK_TFLOPS["bf16"] * 1e12)
        least += max(mem, flop)
        mem_s += mem
    print(json.dumps({
        "metric": f"generated tok/s, {workload} workload, bf16", "value": round(new / dt, 1), "unit": "tokens/s",
        "n_gpus": 1, "seconds": round(dt, 3), "engine_steps": eng.steps - steps0, "higher_is_better": True,
        "vs_reference_published": round(new / dt / w["reference_tok_s"], 2) if "reference_tok_s" in w else None,
        "roofline": {"bound": "hbm or mfma, step by step", "least_seconds": round(least, 3),
                     "least_seconds_memory_alone": round(mem_s, 3), "frac": round(least / dt, 4)},
        "dtype": "bf16", "data": "synthetic: seeded random weights, uniform random token ids",
        "config": {"model": w["name"], "layers": cfg.num_hidden_layers, "layers_of_model": full, "requests": n,
                   "prompt_tokens": sum(lens), "new_tokens": new, "prefill_chunk": w["chunk"],
                   "preemptions": eng.num_preemptions, "total_tok_per_s": round((sum(lens) + new) / dt, 1)}}), flush=True)
    return 0


def product(spec: str, dev="cuda:0") -> int:
    """One bfloat16 product x [M, K] @ w [N, K]^T alone: the many-row tiled kernel (with `slices` of K as
    float32 partial sums, in tile `shape`; left out: what `kernels.tile_split_plan` chooses, or one slice
    in the shape of fewest tiles) beside the vendor library's plain product, each the best of 5 runs of 20
    launches in a HIP graph."""
    import torch
    from xinfer_amd import kernels
    parts = [int(v) for v in spec.split(",")]
    M, N, K = parts[:3]
    slices, shape = (parts[3], parts[4] if len(parts) > 4 else None) if len(parts) > 3 else kernels.tile_split_plan(M, N, K)
    g = torch.Generator(device=dev)
    g.manual_seed(3)
    x = torch.randn((M, K), generator=g, device=dev, dtype=torch.float32).to(torch.bfloat16)
    w = (torch.randn((N, K), generator=g, device=dev, dtype=torch.float32) * 0.05).to(torch.bfloat16)

    def timed(f, n=20):
        f()
        torch.cuda.synchronize()
        graph = torch.cuda.CUDAGraph()
        with torch.cuda.graph(graph):
            for _ in range(n):
                f()
        best = None
        for _ in range(5):
            a, b = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
            a.record()
            graph.replay()
            b.record()
            torch.cuda.synchronize()
            ms = a.elapsed_time(b) / n
            best = ms if best is None else min(best, ms)
        return best * 1e3

    tile_us = timed(lambda: kernels.linear_tile(x, w, slices, partial=slices > 1, shape=shape))
    lib_us = timed(lambda: torch.nn.functional.linear(x, w))
    y = kernels.linear_tile(x, w, slices, partial=slices > 1, shape=shape)
    y = y.sum(0) if y.dim() == 3 else y.float()
    ref = x.float() @ w.float().t()
    flops = 2.0 * M * N * K
    print(json.dumps({"product": [M, N, K], "slices": slices, "tile_shape": shape, "linear_tile_us": round(tile_us, 1),
                      "library_us": round(lib_us, 1), "linear_tile_tflops": round(flops / tile_us / 1e6, 1),
                      "library_tflops": round(flops / lib_us / 1e6, 1),
                      "max_error_of_largest": float((y - ref).abs().max() / ref.abs().max())}), flush=True)
    return 0


def design_compare(spec: str, layers, steps: int, warmup: int, batch: int, context: int, prefill_tokens: int,
                   family: str = "both", only: str = "all") -> int:
    """Mufenex beside Qwen3, Lilalorn, Debusun or Tisosun beside Mufenex, or Vuzazen or Litizen beside Debusun, at equal sizes: ms of the
    prefill of one prompt and of a decode step."""
    import torch
    from xinfer_amd.engine import ModelRunner, StepEntry, build_model
    from xinfer_amd.models import config_from_dict
    from xinfer_amd.sampling import Sampler
    from xinfer_amd.weights.random_init import random_store_for
    name, _, size = spec.partition(":")
    if name not in DESIGN_CHOICES or (size and size not in DESIGN_CHOICES[name][0]):
        print("bench.py: --design " + " or ".join(f"{k}[:{'|'.join(v[0])}]" for k, v in DESIGN_CHOICES.items()))
        return 2
    beside = DESIGN_CHOICES[name][1]
    if family not in ("both", name, beside):
        print(f"bench.py: --family both, {name} or {beside} with --design {name}")
        return 2
    dev, page = "cuda:0", 64
    layers = layers or 4
    sampler = Sampler(dev)
    gen = torch.Generator().manual_seed(3)
    out = {"metric": f"{name.capitalize()} beside {beside.capitalize()} at equal sizes, bf16", "unit": "ms", "layers": layers, "batch": batch,
           "context": context, "prefill_tokens": prefill_tokens, "data": "synthetic: seeded random weights and token ids",
           "sizes": {}}

    def configs(z):
        mixer = dict(dim=z["dim"], heads=z["heads"], kv_heads=z["kv_heads"], vdim=z["vdim"], scale=z["dim"] ** -0.5,
                     softcap=50.0, mask={"size": z["window"]}, v_mix=True)
        mlp = ({"kind": "dense", "ff": z["ff"]} if not z["experts"] else
               {"kind": "moe", "expert": {"ff": z["ff"] // z["top"]}, "router": {"experts": z["experts"], "top": z["top"]}})
        mufenex = {"architecture": "Mufenex", "vocab": DESIGN_VOCAB, "width": z["width"], "embedding": {"scale": 1.0},
                   "norm": {"eps": 1e-6}, "logit_softcap": 30.0, "max_positions": 2 * context,
                   "layers": [{"type": "attention", "mixer": mixer, "mlp": mlp} for _ in range(layers)]}
        qwen3 = dict(QWEN3_8B, hidden_size=z["width"], intermediate_size=z["ff"], num_hidden_layers=layers,
                     num_attention_heads=z["heads"], num_key_value_heads=z["kv_heads"], head_dim=z["dim"],
                     vocab_size=DESIGN_VOCAB, sliding_window=z["window"], max_position_embeddings=2 * context)
        if name == "mufenex":
            return {"mufenex": mufenex, "qwen3": qwen3}
        if name == "tisosun":
            # attention within chunks beside linear attention, a real-gated recurrence, the same again, a minGRU, in turn
            sh = max(1, z["heads"] // 4)
            par = {"left": dict(heads=z["heads"], kv_heads=z["kv_heads"], dim=z["dim"], vdim=z["vdim"], scale=z["dim"] ** -0.5,
                                softcap=50.0, mask={"size": z["window"]},
                                rot=dict(dims=z["dim"] // 2, base=500000.0,
                                         scaling=dict(factor=8.0, original=8192, fast=32.0, slow=1.0))),
                   "right": dict(heads=sh, dim=z["dim"], vdim=2 * z["dim"], decay=[0.95 + 0.049 * h / max(1, sh - 1) for h in range(sh)])}
            kinds = [("parallel", par), ("rglru", dict(width=z["width"], blocks=z["heads"], conv=TISOSUN_TAPS)), ("parallel", par),
                     ("mingru", dict(width=z["width"]))]
            tisosun = {"architecture": "Tisosun", "vocab": DESIGN_VOCAB, "width": z["width"], "norm": {"eps": 1e-6},
                       "token_side": {"dim": TISOSUN_SIDE}, "max_positions": 2 * context,
                       "layers": [{"type": kinds[i % 4][0], "mixer": kinds[i % 4][1], "mlp": mlp} for i in range(layers)]}
            return {"tisosun": tisosun, "mufenex": mufenex}
        if name in ("debusun", "vuzazen", "litizen"):
            # layers of a latent, windowed attention, a state space and windowed attention again, in turn; all of them
            # are one span that runs once, so that the start of a pass is in the step
            rot = dict(dims=z["dim"], base=500000.0)
            lat = dict(heads=z["heads"], dim=z["dim"], vdim=z["vdim"], scale=(z["dim"] + DEBUSUN_LATENT["rot_dim"]) ** -0.5,
                       mask={"size": z["window"]}, **DEBUSUN_LATENT,
                       rot=dict(dims=DEBUSUN_LATENT["rot_dim"], base=500000.0,
                                scaling=dict(factor=8.0, original=8192, fast=32.0, slow=1.0)))
            att = dict(heads=z["heads"], kv_heads=z["kv_heads"], dim=z["dim"], vdim=z["vdim"], scale=z["dim"] ** -0.5,
                       mask={"size": z["window"]}, rot=rot)
            ssm = dict(heads=2 * z["width"] // DEBUSUN_STATE["vdim"], **DEBUSUN_STATE)
            kinds = [("latent_attention", lat), ("attention", att), ("mamba2", ssm), ("attention", att)]
            debusun = {"architecture": "Debusun", "vocab": DESIGN_VOCAB, "width": z["width"], "norm": {"eps": 1e-6},
                       "embedding": {"scale": 1.0, "bigram": {"buckets": 65521, "mul_prev": 1000003, "mul_cur": 31}},
                       "max_positions": 2 * context, "loop": {"start": 0, "stop": layers, "times": 1},
                       "layers": [{"type": kinds[i % 4][0], "mixer": kinds[i % 4][1], "mlp": {"kind": "dense", "ff": z["ff"]}}
                                  for i in range(layers)]}
            if name == "litizen":
                # windowed attention, a state space, attention within chunks, a state space, in turn
                sizes = dict(heads=z["heads"], kv_heads=z["kv_heads"], dim=z["dim"], vdim=z["vdim"], scale=z["dim"] ** -0.5,
                             mask={"size": z["window"]})
                lkinds = [("attention", dict(sizes, rot=rot)), ("mamba2", ssm),
                          ("attention_2", dict(sizes, softcap=50.0, rot=dict(dims=z["dim"] // 2, base=500000.0))), ("mamba2", ssm)]
                lmlp = mlp
                if z["experts"]:
                    lmlp = dict(mlp, router=dict(mlp["router"], identity=LITIZEN_IDENTITY), shared=dict(mlp["expert"]))
                litizen = {"architecture": "Litizen", "vocab": DESIGN_VOCAB, "width": z["width"],
                           "norm": {"eps": 1e-6, "groups": LITIZEN_GROUPS}, "canon": {"taps": LITIZEN_TAPS},
                           "embedding": {"scale": 1.0}, "logit_softcap": 30.0, "max_positions": 2 * context,
                           "layers": [{"type": lkinds[i % 4][0], "mixer": lkinds[i % 4][1], "mlp": lmlp} for i in range(layers)]}
                return {"litizen": litizen, "debusun": debusun}
            if name == "debusun":
                return {"debusun": debusun, "mufenex": mufenex}
            # Vuzazen: a latent, a memory, attention behind a convolution with mixed heads, a memory, in turn; no windows
            vlat = dict(heads=z["heads"], dim=z["dim"], vdim=z["vdim"], q_rank=3 * z["width"] // 8,
                        scale=(z["dim"] + VUZAZEN_LATENT["rot_dim"]) ** -0.5, **VUZAZEN_LATENT,
                        rot=dict(dims=VUZAZEN_LATENT["rot_dim"], base=500000.0))
            vatt = dict(heads=z["heads"], kv_heads=z["kv_heads"], dim=z["dim"], vdim=z["vdim"], scale=z["dim"] ** -0.5, conv=VUZAZEN_TAPS)
            mem = dict(heads=max(1, z["heads"] // 4), dim=z["dim"], vdim=2 * z["dim"], gate_cap=15.0)
            vkinds = [("latent_attention", vlat), ("mlstm", mem), ("attention", vatt), ("mlstm", mem)]
            vuzazen = {"architecture": "Vuzazen", "vocab": DESIGN_VOCAB, "width": z["width"], "norm": {"eps": 1e-6},
                       "embedding": {"scale": 1.0, "bigram": {"buckets": 65521, "mul_prev": 1000003, "mul_cur": 31}},
                       "max_positions": 2 * context,
                       "layers": [{"type": vkinds[i % 4][0], "mixer": vkinds[i % 4][1], "mlp": mlp} for i in range(layers)]}
            return {"vuzazen": vuzazen, "debusun": debusun}
        # Lilalorn: layers of attention beside retention and of gated linear attention in turn; the states' heads are a
        # quarter as many as the query heads, keys as wide as the attention's and values twice that
        mixer.pop("mask")
        mixer["v_mix"] = False
        sh = max(1, z["heads"] // 4)
        moe = {"kind": "moe", "expert": {"ff": z["ff"] // z["top"]}, "router": {"experts": z["experts"], "top": z["top"]},
               "shared": {"ff": z["ff"] // z["top"]}}
        par = {"type": "parallel", "mlp": moe, "mixer": {
            "left": dict(heads=z["heads"], kv_heads=z["kv_heads"], dim=z["dim"], vdim=z["vdim"], scale=z["dim"] ** -0.5,
                         rot=dict(dims=z["dim"], base=500000.0, scaling=dict(factor=8.0, low=1.0, high=4.0, original=8192))),
            "right": dict(heads=sh, dim=z["dim"], vdim=2 * z["dim"], decay=[0.95 + 0.049 * h / max(1, sh - 1) for h in range(sh)]),
            "left_scale": 0.75, "right_scale": 0.4}}
        gla = {"type": "gla", "mlp": moe, "mixer": dict(heads=sh, dim=z["dim"], vdim=2 * z["dim"], tau=8.0)}
        lilalorn = {"architecture": "Lilalorn", "vocab": DESIGN_VOCAB, "width": z["width"], "norm": {"eps": 1e-6},
                    "residual_mult": 0.8, "logit_scale": 0.25, "max_positions": 2 * context,
                    "layers": [par if i % 2 == 0 else gla for i in range(layers)]}
        return {"lilalorn": lilalorn, "mufenex": mufenex}

    def time_model(raw):
        _, cfg = config_from_dict(raw)
        model = build_model(cfg, random_store_for(cfg, seed=0, linear_std=0.02, norm_std=0.1), "bf16", dev)
        pages = batch * (-(-context // page) + 2) + -(-prefill_tokens // page) + 8
        runner = ModelRunner(model, page_size=page, num_pages=pages, max_requests=batch + 1)
        g = torch.Generator(device=dev).manual_seed(1)
        for lc in runner.layer_caches.values():
            for t in lc.pools.values():
                t.copy_(torch.randn(t.shape, generator=g, device=dev, dtype=torch.float32).to(t.dtype))
        vocab = model.spec.vocab_size
        ids = torch.randint(0, vocab, (prefill_tokens,), generator=gen).tolist()
        best = None
        for _ in range(4 if only != "decode" else 0):      # the first run warms up
            runner.add_request(7)
            torch.cuda.synchronize()
            t = time.perf_counter()
            sampler.argmax(runner.step([StepEntry(7, ids, [prefill_tokens - 1])])).tolist()
            torch.cuda.synchronize()
            dt = time.perf_counter() - t
            runner.release(7)
            best = dt if best is None else min(best, dt)
        if only == "prefill":
            return {"prefill_ms": round(best * 1e3, 3), "prefill_tok_s": round(prefill_tokens / best, 1)}
        prep = runner.graph_after
        start = context - steps - warmup - prep
        rids = list(range(100, 100 + batch))
        for rid in rids:
            runner.add_request(rid)
            runner.cache.reserve(rid, start)
            runner.cache.commit(rid, start)
        places = list(range(batch))
        prev = None

        def one(prev):
            if prev is None:
                toks = torch.randint(0, vocab, (batch,), generator=gen).tolist()
                logits = runner.step([StepEntry(r, [t], [0]) for r, t in zip(rids, toks)])
            else:
                logits = runner.step([StepEntry(r, [0], [0]) for r in rids], device_tokens=(prev, places, places))
            return sampler.argmax(logits)
        for _ in range(prep + warmup):
            prev = one(prev)
        torch.cuda.synchronize()
        t = time.perf_counter()
        for _ in range(steps):
            prev = one(prev)
        torch.cuda.synchronize()
        dec = (time.perf_counter() - t) / steps
        assert 0 <= int(prev.min()) and int(prev.max()) < vocab
        replays = runner.graph_replays
        del runner, model
        torch.cuda.empty_cache()
        res = {"decode_ms": round(dec * 1e3, 4), "decode_tok_s": round(batch / dec, 1), "graph_replays": replays}
        if best is not None:
            res.update({"prefill_ms": round(best * 1e3, 3), "prefill_tok_s": round(prefill_tokens / best, 1)})
        return res

    for key in ([size] if size else list(DESIGN_CHOICES[name][0])):
        z = DESIGN_SIZES[key]
        res = {k: time_model(raw) for k, raw in configs(z).items() if family in ("both", k)}
        for what in ("prefill", "decode"):
            if family == "both" and f"{what}_ms" in res[name]:
                res[f"ratio_{what}"] = round(res[name][f"{what}_ms"] / res[beside][f"{what}_ms"], 3)
        out["sizes"][key] = dict(z, **res)
        print(f"[bench] {key}: {res}", file=sys.stderr, flush=True)
    print(json.dumps(out), flush=True)
    return 0


def measured_peaks(dev="cuda:0"):
    """(GB/s of a read-only stream over 4 GiB, TFLOP/s of one square bfloat16 product of 8192 in the
    vendor library): what this card reaches, beside the published peaks.  Best of five runs each."""
    import torch
    from xinfer_amd import kernels
    buf = torch.empty(1 << 30, dtype=torch.int32, device=dev)         # 4 GiB: sixteen times the memory-side cache
    buf.zero_()
    best = None
    for workgroups, chunk in ((256, 1 << 18), (256, 1 << 16), (1024, 1 << 14)):     # the shapes that read fastest
        for _ in range(5):
            a, b = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
            a.record()
            kernels.stream_read(buf, workgroups, chunk)
            b.record()
            torch.cuda.synchronize()
            ms = a.elapsed_time(b)
            best = ms if best is None else min(best, ms)
    gbps = buf.numel() * 4 / (best * 1e-3) / 1e9
    del buf
    n = 8192
    x = torch.randn(n, n, device=dev, dtype=torch.float32).to(torch.bfloat16)
    w = torch.randn(n, n, device=dev, dtype=torch.float32).to(torch.bfloat16)
    best = None
    for _ in range(6):
        a, b = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
        a.record()
        torch.nn.functional.linear(x, w)
        b.record()
        torch.cuda.synchronize()
        ms = a.elapsed_time(b)
        best = ms if best is None else min(best, ms)
    tflops = 2.0 * n * n * n / (best * 1e-3) / 1e12
    return gbps, tflops


def main() -> int:
    global CONTEXT, PREFILL_TOKENS
    ap = argparse.ArgumentParser()
    ap.add_argument("--gpus", type=int, default=1)
    ap.add_argument("--steps", type=int, default=64)
    ap.add_argument("--warmup", type=int, default=8)
    ap.add_argument("--layers", type=int, default=None,
                    help="fewer layers than the configuration has (reported in config)")
    ap.add_argument("--workload", choices=["decode"] + sorted(WORKLOADS), default="decode",
                    help="decode: the contract's run (default); the others: a serving workload end to end")
    ap.add_argument("--batch", type=int, default=8)
    ap.add_argument("--context", type=int, default=CONTEXT,
                    help="context length at the end of the decode run (default: the contract's)")
    ap.add_argument("--prefill-tokens", type=int, default=PREFILL_TOKENS,
                    help="length of the prefilled prompt (default: the contract's)")
    ap.add_argument("--model", choices=sorted(MODELS), default="8b",
                    help="layer sizes of the decode and prefill runs (default: the contract's Qwen3-8B)")
    ap.add_argument("--skip-points", action="store_true", help="only the default decode run")
    ap.add_argument("--only", choices=["all", "decode", "prefill"], default="all",
                    help="run one phase only (for profiling); the JSON line then lacks the other")
    ap.add_argument("--no-run-ahead", action="store_true",
                    help="serving workloads: read every step's tokens on the host before the next step is planned")
    ap.add_argument("--product", default=None, metavar="M,N,K[,slices[,shape]]",
                    help="time one bfloat16 product alone in the many-row tiled kernel and in the vendor library")
    ap.add_argument("--design", default=None, metavar="mufenex[:SIZE]|lilalorn[:SIZE]|debusun[:SIZE]|litizen[:SIZE]|tisosun[:SIZE]|vuzazen[:SIZE]",
                    help="time another model family beside its closest one (Mufenex beside Qwen3, Lilalorn, Debusun or Tisosun beside Mufenex, Vuzazen or Litizen beside Debusun) at equal sizes (a line of its own; --layers, --steps, "
                         "--warmup, --batch, --context, --prefill-tokens and --only apply)")
    ap.add_argument("--family", choices=["both", "debusun", "lilalorn", "litizen", "mufenex", "qwen3", "tisosun", "vuzazen"], default="both",
                    help="--design: time one of the two families only (for profiling)")
    ap.add_argument("--peaks", action="store_true",
                    help="also measure what this card reaches on a read-only stream of 4 GiB and on one square "
                         "bfloat16 product of 8192, and report the fractions of those beside the fractions of the "
                         "published peaks")
    args = ap.parse_args()
    if args.gpus != 1:
        print(f"bench.py: this engine runs on one GPU; --gpus {args.gpus} is not supported")
        return 2
    if args.product:
        return product(args.product)
    if args.design:
        return design_compare(args.design, args.layers, args.steps, args.warmup, args.batch, args.context, args.prefill_tokens,
                              args.family, args.only)
    if args.workload != "decode":
        return serve(args.workload, args.layers, not args.no_run_ahead)
    full_layers = MODELS[args.model]["num_hidden_layers"]
    model_name = {"0.6b": "Qwen3-0.6B", "8b": "Qwen3-8B", "14b": "Qwen3-14B", "32b": "Qwen3-32B"}[args.model]
    if args.layers is None:
        args.layers = full_layers
    CONTEXT, PREFILL_TOKENS = args.context, args.prefill_tokens     # the sizes of this run

    import torch
    from xinfer_amd.engine import ModelRunner, StepEntry, build_model
    from xinfer_amd.models import config_from_dict
    from xinfer_amd.sampling import Sampler
    from xinfer_amd.weights.random_init import random_store_for

    dev = "cuda:0"
    raw = dict(MODELS[args.model], num_hidden_layers=args.layers)
    _, cfg = config_from_dict(raw)
    store = random_store_for(cfg, seed=0, linear_std=0.02, norm_std=0.1)
    t0 = time.time()
    model = build_model(cfg, store, "bf16", dev)
    torch.cuda.synchronize()
    print(f"[bench] model of {args.layers} layers built in {time.time() - t0:.1f}s", file=sys.stderr, flush=True)

    page = 64
    max_batch = 8 if (args.skip_points or args.only != "all") else 64
    max_batch = max(max_batch, args.batch)
    num_pages = max_batch * (-(-CONTEXT // page)) + -(-PREFILL_TOKENS // page) + 8
    runner = ModelRunner(model, page_size=page, num_pages=num_pages, max_requests=max_batch + 1)
    g = torch.Generator(device=dev)
    g.manual_seed(1)
    for lc in runner.layer_caches.values():          # random cache contents for the decode runs
        lc.k.copy_(torch.randn(lc.k.shape, generator=g, device=dev, dtype=torch.float32).to(lc.k.dtype))
        lc.v.copy_(torch.randn(lc.v.shape, generator=g, device=dev, dtype=torch.float32).to(lc.v.dtype))
    sampler = Sampler(dev)
    cpu_gen = torch.Generator().manual_seed(2)

    def sync():
        torch.cuda.synchronize()

    def decode_run(batch, steps, warmup, context=None):
        """`batch` requests whose caches already hold context - steps - warmup tokens decode
        steps + warmup tokens, so that the last timed step ends at `context` (CONTEXT unless given)."""
        prep = runner.graph_after          # steps before the warm-up in which the decode graph is recorded
        start = (context or CONTEXT) - steps - warmup - prep
        rids = list(range(100, 100 + batch))
        for rid in rids:
            runner.add_request(rid)
            runner.cache.reserve(rid, start)
            runner.cache.commit(rid, start)
        toks = torch.randint(0, cfg.vocab_size, (batch,), generator=cpu_gen).tolist()
        places = list(range(batch))
        pins = [torch.empty((batch,), dtype=torch.int32, pin_memory=True) for _ in range(2)]
        state = {"turn": 0}

        def one(prev):
            """One decode step as the engine launches it (`LLMEngine.step` with its default
            `run_ahead`): the tokens that the step before sampled are handed over on the device,
            greedy sampling follows on the GPU, and the sampled ids start their way to the host
            without anything waiting for them; the host prepares the next step meanwhile."""
            if prev is None:
                logits = runner.step([StepEntry(r, [t], [0]) for r, t in zip(rids, toks)])
            else:
                logits = runner.step([StepEntry(r, [0], [0]) for r in rids], device_tokens=(prev, places, places))
            tok = sampler.argmax(logits)
            pins[state["turn"]].copy_(tok, non_blocking=True)
            state["turn"] ^= 1
            return tok

        prev = None
        for _ in range(prep + warmup):
            prev = one(prev)
        sync()
        t = time.perf_counter()
        for _ in range(steps):
            prev = one(prev)
        sync()
        dt = time.perf_counter() - t
        assert 0 <= int(prev.min()) and int(prev.max()) < cfg.vocab_size
        for rid in rids:
            runner.release(rid)
        return dt / steps

    def prefill_run(reps=3):
        ids = torch.randint(0, cfg.vocab_size, (PREFILL_TOKENS,), generator=cpu_gen).tolist()
        best = None
        for _ in range(reps + 1):                  # the first run warms up
            runner.add_request(7)
            sync()
            t = time.perf_counter()
            logits = runner.step([StepEntry(7, ids, [PREFILL_TOKENS - 1])])
            sampler.argmax(logits).tolist()
            sync()
            dt = time.perf_counter() - t
            runner.release(7)
            best = dt if best is None else min(best, dt)
        return best

    if args.only == "prefill":
        psec = prefill_run()
        print(json.dumps({"prefill_ms": round(psec * 1e3, 3), "layers": args.layers}), flush=True)
        return 0
    sec = decode_run(args.batch, args.steps, args.warmup)
    wb, kvb = weight_bytes(cfg), kv_bytes_per_token(cfg)

    def stream_rate(batch, steps, seconds, context):
        """GB/s of a decode step: every weight once and the cache of its requests, over its time.  The
        cache length is the mean over the timed steps (it grows by one a step and ends at `context`)."""
        return (wb + batch * (context - (steps - 1) / 2.0) * kvb) / seconds / 1e9

    achieved = stream_rate(args.batch, args.steps, sec, CONTEXT)
    out = {
        "metric": f"decode tok/s at batch {args.batch}, {model_name} bf16", "value": round(args.batch / sec, 2),
        "unit": "tokens/s", "n_gpus": 1, "steps": args.steps, "warmup": args.warmup,
        "ms_per_step": round(sec * 1e3, 4), "higher_is_better": True, "scaling": "weak",
        "vs_baseline": None, "dtype": "bf16",
        "data": "synthetic: seeded random weights, uniform random token ids, random cache contents",
        "config": {
            "model": f"{model_name} layer sizes", "global_batch": args.batch, "seq_len": CONTEXT,
            "parallelism": "single GPU", "layers": args.layers, "layers_of_model": full_layers,
            "hidden_size": cfg.hidden_size, "intermediate_size": cfg.intermediate_size,
            "num_attention_heads": cfg.num_attention_heads, "num_key_value_heads": cfg.num_key_value_heads,
            "head_dim": cfg.head_dim, "vocab_size": cfg.vocab_size, "rope_theta": cfg.rope_theta,
            "rms_norm_eps": cfg.rms_norm_eps, "tie_word_embeddings": cfg.tie_word_embeddings,
            "page_size": page, "prefill_tokens": PREFILL_TOKENS, "kv_dtype": "bf16"},
        "roofline": {"bound": "hbm", "achieved": round(achieved, 1), "peak": HBM_GBPS, "unit": "GB/s",
                     "frac": round(achieved / HBM_GBPS, 4)},
    }
    print(f"[bench] decode b{args.batch}: {sec * 1e3:.3f} ms/step", file=sys.stderr, flush=True)
    peaks = None
    if args.peaks:
        peaks = measured_peaks(dev)
        out["peaks_measured"] = {"hbm_read_GBps": round(peaks[0], 1), "bf16_product_TFLOPs": round(peaks[1], 1)}
        out["roofline"]["frac_of_measured"] = round(achieved / peaks[0], 4)
        print(f"[bench] measured peaks: {peaks[0]:.0f} GB/s read-only stream, {peaks[1]:.0f} TFLOP/s square bf16 product",
              file=sys.stderr, flush=True)
    if args.only == "decode":
        print(json.dumps(out), flush=True)
        return 0
    psec = prefill_run()
    flops = prefill_flops(cfg, PREFILL_TOKENS)
    out["prefill"] = {"value": round(PREFILL_TOKENS / psec, 1), "tokens": PREFILL_TOKENS,
                      "ms": round(psec * 1e3, 3),
                      "frac": round(flops / psec / (PEAK_TFLOPS["bf16"] * 1e12), 4)}
    if peaks is not None:
        out["prefill"]["frac_of_measured"] = round(flops / psec / (peaks[1] * 1e12), 4)
    print(f"[bench] prefill {PREFILL_TOKENS}: {psec * 1e3:.2f} ms", file=sys.stderr, flush=True)
    if not args.skip_points:
        points, roofs = {}, {}
        k, w = max(8, args.steps // 2), max(2, args.warmup // 2)
        for b in (1, 64):
            s = decode_run(b, k, w)
            points[f"decode_b{b}"] = round(b / s, 2)
            rate = stream_rate(b, k, s, CONTEXT)
            roofs[f"decode_b{b}"] = {"ms_per_step": round(s * 1e3, 4), "achieved": round(rate, 1),
                                     "frac": round(rate / HBM_GBPS, 4)}
            print(f"[bench] decode b{b}: {s * 1e3:.3f} ms/step", file=sys.stderr, flush=True)
        out["points"] = points
        out["points_roofline"] = roofs          # GB/s of each point's step and its fraction of the 8 TB/s peak
        # one point at a longer context: batch 8 with 16,384 tokens in every request's cache
        far = 4 * CONTEXT
        if max_batch * (-(-CONTEXT // page)) >= 8 * (-(-far // page)) and far <= cfg.max_position_embeddings:
            s = decode_run(8, k, w, context=far)
            rate = stream_rate(8, k, s, far)
            out["further"] = {"decode_b8_ctx": far, "value": round(8 / s, 2), "ms_per_step": round(s * 1e3, 4),
                              "achieved": round(rate, 1), "frac": round(rate / HBM_GBPS, 4)}
            print(f"[bench] decode b8 at context {far}: {s * 1e3:.3f} ms/step", file=sys.stderr, flush=True)
    print(json.dumps(out), flush=True)
    return 0


if __name__ == "__main__":
    sys.exit(main())
