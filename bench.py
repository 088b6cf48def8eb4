#!/usr/bin/python3
"""Measurement: GPT-2 XL shape, random weights, on one MI355X.

    python bench.py [--gpus 1] [--steps K] [--warmup W]

A step is one decode step of the engine (scheduler, step function, sampling): batch 8 from a
512-token context by default.  Every figure is the median of three blocks of K steps (of three runs for
the prefill).  One JSON line: decoded tokens a second, the prefill of 2,048 tokens (two prompts of 1,024
in one step), the decode step's share of the HBM roofline, decoding at batch 1 and 64 (`points`: tokens a
second; `point_details`: milliseconds, bytes and share of the roofline of each), and the 32-bit engine's
decode steps and prefill (`fp32`).  Peaks are the published ones of MI355X.

    python bench.py --only decode|prefill [--kernel-times]   one workload; with --kernel-times kernel by
                                                             kernel, each launch between two HIP events
    python bench.py --only serving [--dtype float32]         BASELINE.json's configs[3] through the scheduler
    python bench.py --only replay [--sequences 8] [--shape xl]   BASELINE.json's configs[4] (or configs[2]'s sizes)
                                                             against the plain implementation, in four ways of cutting
    python bench.py --only ridopel [--width 1024] [--kernel-times]   four Ridopel layers (latent attention, hgrn2, latent
                                                             attention, wkv, each with sixteen experts) beside four GPT-2
                                                             layers of the same width: prefill and decode
    python bench.py --only pafivik [--width 1024] [--kernel-times]   four Pafivik layers (lightning, channel_delta, attention,
                                                             channel_delta, each with sixteen experts and a shared one) beside
                                                             four Ridopel layers of the same width: prefill and decode
    python bench.py --only dogalorn [--width 1024] [--kernel-times]  four Dogalorn layers (attention in chunks beside a minGRU,
                                                             Mamba2, Mamba2, the pair again; dense feed-forwards; the stream in two
                                                             copies) beside four Pafivik layers with dense feed-forwards of the same
                                                             width (attention, lightning, lightning, attention): prefill and decode
    python bench.py --only nigilorn [--width 1024] [--kernel-times]  four Nigilorn layers (selective scan, attention in a window,
                                                             latent attention in a window, selective scan; a dense feed-forward, then
                                                             sixteen experts and a shared one; gated sublayers, a token input behind
                                                             every layer) beside four Pafivik layers of the same width and feed-forward
                                                             sizes (lightning, attention, attention, lightning): prefill and decode
    python bench.py --only fikupel [--width 1024] [--kernel-times]   four Fikupel layers (attention in a window that keeps first tokens,
                                                             latent attention in a window, both again; a dense feed-forward, then
                                                             sixteen experts; the stream in four copies) beside four Nigilorn layers
                                                             of the same kinds and sizes: prefill and decode
    python bench.py --only pepapel [--width 1024] [--kernel-times]   four Pepapel layers (a pair of attention in chunks and a delta rule,
                                                             attention with a soft cap, the pair twice; a dense feed-forward, then
                                                             sixteen experts and four outputs that return their input) beside
                                                             seven Pafivik layers that hold the same mixers and as many
                                                             feed-forwards: prefill and decode
"""
import argparse
import json
import os
import statistics
import sys
import time

ROOT = os.path.dirname(os.path.abspath(__file__))
sys.path.insert(0, ROOT)

HBM_PEAK_GBS = 8000.0
MFMA_PEAK = {"bf16": 2.5e15, "fp32": 157.3e12}
SHORT = {"bfloat16": "bf16", "float32": "fp32"}


def baseline_config(index, n_layer=0):
    """The sizes that BASELINE.json's configs[index] names in words -> (config.json keys, its layers)."""
    import re
    with open(os.path.join(ROOT, "BASELINE.json")) as f:
        text = json.load(f)["configs"][index]
    num = lambda key: int(re.search(key + r"=(\d+)", text).group(1))   # noqa: E731
    cfg = dict(architectures=["GPT2LMHeadModel"], n_layer=num("n_layer"), n_embd=num("n_embd"), n_head=num("n_head"),
               n_inner=num("n_inner"), vocab_size=num("vocab_size"), n_positions=num("n_positions"),
               layer_norm_epsilon=1e-5, activation_function="gelu_new")
    full = cfg["n_layer"]
    if n_layer:
        cfg["n_layer"] = n_layer
    return cfg, full


class Workloads:
    """The decode and prefill measurements on one runner."""

    def __init__(self, a, dtype, cfg=None):
        """cfg: a config.json of any architecture with the keys n_positions and vocab_size beside its own (default:
        the shape that --shape names)."""
        import torch
        from denno_beta_amd.config import EngineOptions
        from denno_beta_amd.engine import ModelRunner
        self.torch, self.a, self.dtype = torch, a, dtype
        if cfg is None:
            self.cfg, self.full_layers = baseline_config({"xl": 2, "large": 3, "medium": 4}[a.shape], a.layers)
        else:
            self.cfg, self.full_layers = cfg, 0
        P = self.cfg["n_positions"]
        live = max(64, a.batch)
        self.opts = EngineOptions(dtype=dtype, page_size=a.page_size, cache_tokens=live * P, max_live=live, max_batch_tokens=4096,
                                  prefill_chunk=1024, use_graphs=not (a.no_graphs or a.kernel_times), seed=0,
                                  norms_inside_products=not a.norm_kernels, deferred_sums=not a.no_deferred_sums)
        self.runner = ModelRunner.from_random(self.cfg, seed=0, options=self.opts, stored=dtype)
        self.gen = torch.Generator().manual_seed(0)

    def prompt(self, n):
        return self.torch.randint(0, self.cfg["vocab_size"], (n,), generator=self.gen).tolist()

    def decode(self, batch, steps, warmup, blocks=3, on_start=None):
        """-> {ms, tok_s, bytes, frac, mean_context}: the median block of `steps` steps.  on_start: called once the
        prompts are in the cache and the warm-up steps are done, before the first timed step."""
        from denno_beta_amd.engine import Engine, SamplingParams
        a, P, sync = self.a, self.cfg["n_positions"], self.torch.cuda.synchronize
        steps = max(1, min(steps, (P - a.context - warmup - 2) // blocks))
        eng = Engine(self.runner, self.opts)
        # greedy, unless --only decode names other sampling options (what the sampling kernels cost a step)
        sp = SamplingParams(max_tokens=P, temperature=getattr(a, "temperature", 0.0), top_k=getattr(a, "top_k", None),
                            top_p=getattr(a, "top_p", None), repetition_penalty=getattr(a, "repetition_penalty", None),
                            seed=3, ignore_eos=True)
        rids = [eng.add_request(self.prompt(a.context), sp) for _ in range(batch)]
        while any(eng.scheduler.computed(r) < a.context for r in rids):
            eng.step()
        for _ in range(warmup):
            eng.step()
        if on_start is not None:
            sync()
            on_start()
        times = []
        for _ in range(blocks):
            sync()
            t0 = time.perf_counter()
            for _ in range(steps):
                eng.step()
            sync()
            times.append((time.perf_counter() - t0) / steps)
        assert all(len(eng.requests[r].generated) >= blocks * steps for r in rids)
        for r in rids:
            eng.abort(r)
        order = sorted(range(blocks), key=lambda i: times[i])
        mid = order[blocks // 2]
        mean_ctx = a.context + 1 + warmup + mid * steps + (steps - 1) / 2.0
        nbytes = self.runner.model.weight_bytes() + batch * mean_ctx * self.runner.cache.bytes_per_token()
        t = times[mid]
        return {"ms": t * 1e3, "tok_s": batch / t, "bytes": nbytes, "frac": nbytes / t / 1e9 / HBM_PEAK_GBS,
                "mean_context": mean_ctx, "steps": steps}

    def prefill(self, reps=3, prompts=2):
        """-> {value, tokens, ms, frac}: `prompts` prompts of 1,024 tokens in one step (two: the 2,048 tokens
        of the contract), the median of `reps`."""
        from denno_beta_amd.engine import StepEntry
        runner, sync = self.runner, self.torch.cuda.synchronize
        times = []
        for i in range(reps + 1):
            seqs = [self.prompt(1024) for _ in range(prompts)]
            for j in range(prompts):
                runner.start_request(1000 + j)
            sync()
            t0 = time.perf_counter()
            runner.step([StepEntry(1000 + j, seqs[j], [1023]) for j in range(prompts)])
            sync()
            times.append(time.perf_counter() - t0)
            for j in range(prompts):
                runner.end_request(1000 + j)
        t = statistics.median(times[1:])
        cfg = self.cfg
        V, E = cfg["vocab_size"], cfg.get("n_embd", cfg.get("width"))
        mat = sum(w.numel() for w in _layer_matrices(runner))
        tokens = 1024 * prompts
        flops = 2.0 * tokens * mat + 2.0 * prompts * V * E + cfg.get("n_layer", len(cfg.get("layers", ()))) * prompts * (4.0 * E * 1024 * 1025 / 2)
        return {"value": tokens / t, "tokens": tokens, "ms": t * 1e3, "frac": flops / t / MFMA_PEAK[SHORT[self.dtype]]}


def _layer_matrices(runner):
    from denno_beta_amd.parts import Linear
    seen = []
    for b in runner.model.blocks:
        for p in b.parts():
            for v in vars(p).values():
                if isinstance(v, Linear):
                    seen.append(v.weight)
    return seen


def kernel_table(what):
    """Prints the per-kernel shares that ops.time_launches measured."""
    from denno_beta_amd.kernels import ops
    times = ops.launch_times()
    total = sum(ms for _, ms in times.values())
    print(f"{what}: {total:.3f} ms in {sum(n for n, _ in times.values())} launches (each between two events)")
    for name, (n, ms) in sorted(times.items(), key=lambda kv: -kv[1][1]):
        print(f"  {ms / total * 100:5.1f} %  {ms / n * 1e3:8.1f} us x {n:5d}  {name}")


def main():
    ap = argparse.ArgumentParser()
    ap.add_argument("--gpus", type=int, default=1)
    ap.add_argument("--steps", type=int, default=100)
    ap.add_argument("--warmup", type=int, default=10)
    ap.add_argument("--batch", type=int, default=8)
    ap.add_argument("--context", type=int, default=512)
    ap.add_argument("--dtype", default="bfloat16", choices=["bfloat16", "float32"])
    ap.add_argument("--layers", type=int, default=0, help="fewer layers than the configuration (0: all)")
    ap.add_argument("--no-graphs", action="store_true")
    ap.add_argument("--norm-kernels", action="store_true",
                    help="run every norm as a kernel of its own, also in steps of few rows (for comparisons)")
    ap.add_argument("--no-deferred-sums", action="store_true",
                    help="every product into the stream adds its own sum (steps of 65 to 256 rows; for comparison)")
    ap.add_argument("--no-points", action="store_true", help="skip batch 1 and 64, the prefill and the 32-bit engine")
    ap.add_argument("--kernel-times", action="store_true",
                    help="with --only decode or prefill: every launch between two HIP events (no graphs), and a "
                         "table of each kernel's share")
    ap.add_argument("--sequences", type=int, default=8, help="--only replay: how many of the eight sequences")
    ap.add_argument("--page-size", type=int, default=16, help="tokens in a page of the cache (decode and prefill)")
    ap.add_argument("--prompts", type=int, default=2, help="--only prefill: prompts of 1,024 tokens in the one step")
    ap.add_argument("--temperature", type=float, default=0.0, help="--only decode: sampling instead of greedy (0: greedy)")
    ap.add_argument("--top-k", type=int, default=None, help="--only decode, with --temperature")
    ap.add_argument("--top-p", type=float, default=None, help="--only decode, with --temperature")
    ap.add_argument("--repetition-penalty", type=float, default=None, help="--only decode: penalties over each request's tokens")
    ap.add_argument("--shape", choices=["xl", "large", "medium"], default=None,
                    help="--only decode / prefill / replay: the layer sizes of BASELINE.json's configs[2], [3] or [4] "
                         "(default xl; for replay medium)")
    ap.add_argument("--width", type=int, default=0, help="--only ridopel, pafivik, dogalorn, nigilorn, fikupel, pepapel: one width instead of 1,024 and 2,048")
    ap.add_argument("--only", choices=["decode", "prefill", "serving", "replay", "ridopel", "pafivik", "dogalorn", "nigilorn", "fikupel", "pepapel"], default=None,
                    help="run one workload and print a short line (decode, prefill: for profiling; serving: "
                         "BASELINE.json's configs[3], GPT-2 Large shape, 64 requests through the scheduler; replay: "
                         "configs[4], GPT-2 Medium shape, against the plain implementation)")
    a = ap.parse_args()
    if a.gpus != 1:
        print(f"bench.py: this engine runs on one GPU; --gpus {a.gpus} is not supported")
        sys.exit(2)
    if a.only == "serving":
        return serving(a)
    if a.only == "ridopel":
        return ridopel(a)
    if a.only == "pafivik":
        return pafivik(a)
    if a.only == "dogalorn":
        return dogalorn(a)
    if a.only == "nigilorn":
        return nigilorn(a)
    if a.only == "fikupel":
        return fikupel(a)
    if a.only == "pepapel":
        return pepapel(a)
    if a.only == "replay":
        a.shape = a.shape or "medium"      # (configs[4] as written; --shape xl: the same replay at configs[2]'s sizes)
        return replay(a)
    a.shape = a.shape or "xl"

    if a.only != "decode" and (a.temperature or a.top_k or a.top_p or a.repetition_penalty):
        print("bench.py: sampling options go with --only decode (the contract's line is greedy)")
        sys.exit(2)
    w = Workloads(a, a.dtype)
    if a.only in ("prefill", "decode"):
        from denno_beta_amd.kernels import ops
        if a.only == "prefill":
            w.prefill(1, a.prompts)
            if a.kernel_times:
                ops.time_launches(True)
            r = w.prefill(1 if a.kernel_times else 3, a.prompts)
            print(json.dumps({"prefill_ms": r["ms"], "tokens": r["tokens"], "tok_s": r["value"], "frac": r["frac"]}))
        else:
            if a.kernel_times:
                w.decode(a.batch, 2, 2, blocks=1)
                ops.time_launches(True)
            r = w.decode(a.batch, a.steps, a.warmup, blocks=1 if a.kernel_times else 3)
            print(json.dumps({"decode_ms_per_step": r["ms"], "batch": a.batch, "mean_context": r["mean_context"],
                              "frac": r["frac"]}))
        if a.kernel_times:
            kernel_table(f"{a.only}, {a.dtype}")
        return

    main_point = w.decode(a.batch, a.steps, a.warmup)
    cfg, short = w.cfg, SHORT[a.dtype]
    out = {
        "metric": "GPT-2 XL decode tokens/s (batch 8, context 512)", "value": main_point["tok_s"], "unit": "tokens/s",
        "n_gpus": 1, "steps": main_point["steps"], "warmup": a.warmup, "ms_per_step": main_point["ms"],
        "higher_is_better": True, "scaling": "weak", "vs_baseline": None, "dtype": short, "data": "synthetic",
        "config": {"model": f"gpt2-{a.shape}-shape", "n_layer": cfg["n_layer"], "n_layer_full": w.full_layers,
                   "n_embd": cfg["n_embd"], "n_head": cfg["n_head"], "n_inner": cfg["n_inner"],
                   "vocab_size": cfg["vocab_size"], "n_positions": cfg["n_positions"], "global_batch": a.batch,
                   "seq_len": a.context, "page_size": w.opts.page_size, "weights": "random N(0,0.02)",
                   "graphs": w.opts.use_graphs, "timing": "median of 3 blocks", "parallelism": "single-gpu"},
        "roofline": {"bound": "hbm", "achieved": main_point["bytes"] / main_point["ms"] / 1e6, "peak": HBM_PEAK_GBS,
                     "unit": "GB/s", "frac": main_point["frac"]},
    }
    if not a.no_points:
        out["prefill"] = w.prefill()
        b1 = w.decode(1, min(a.steps, 100), a.warmup)
        b64 = w.decode(64, min(a.steps, 50), a.warmup)
        out["points"] = {"decode_b1": b1["tok_s"], "decode_b64": b64["tok_s"]}
        keep = lambda r: {k: r[k] for k in ("ms", "tok_s", "bytes", "frac")}   # noqa: E731
        out["point_details"] = {"decode_b1": keep(b1), f"decode_b{a.batch}": keep(main_point), "decode_b64": keep(b64)}
        if a.dtype == "bfloat16":
            # the true 32-bit engine at the same sizes: every product in the plain kernels
            del w
            import torch
            torch.cuda.empty_cache()
            f = Workloads(a, "float32")
            f1, f8 = f.decode(1, min(a.steps, 10), 2), f.decode(8, min(a.steps, 10), 2)
            out["fp32"] = {"decode_b1": keep(f1), "decode_b8": keep(f8), "prefill": f.prefill()}
    print(json.dumps(out))


def ridopel_configs(width, layers=4, vocab=32000, positions=2048):
    """-> (a Ridopel config, a GPT-2 config) of the same width, layers, vocabulary and positions.  The Ridopel layers
    take turns between latent attention (heads of 64 + 32, a kept key of 224 + 32 numbers), hgrn2 (heads of 64 keys x 128
    values) and wkv (heads of 64), each with sixteen experts of the model's width of which a token uses two."""
    H = width // 128
    moe = dict(kind="moe", expert=dict(ff=width, limit=7.0), router=dict(experts=16, top=2))
    lat = dict(type="latent_attention", mlp=moe, mixer=dict(heads=H, dim=64, rot_dim=32, vdim=128, kv_rank=224, scale=96 ** -0.5,
                                                            rot=dict(base=10000.0, dims=32)))
    kinds = [lat, dict(type="hgrn2", mlp=moe, mixer=dict(heads=H, dim=64, vdim=128)), lat,
             dict(type="wkv", mlp=moe, mixer=dict(heads=width // 64, dim=64, decay_rank=64))]
    rid = dict(architecture="Ridopel", vocab=vocab, width=width, norm=dict(eps=1e-5), canon=dict(taps=4), logit_softcap=30.0,
               layers=[kinds[i % 4] for i in range(layers)], max_positions=positions, n_positions=positions, vocab_size=vocab)
    gpt = dict(architectures=["GPT2LMHeadModel"], n_layer=layers, n_embd=width, n_head=width // 64, n_inner=4 * width,
               vocab_size=vocab, n_positions=positions, layer_norm_epsilon=1e-5, activation_function="gelu_new")
    return rid, gpt


def pafivik_configs(width, layers=4, vocab=32000, positions=2048):
    """-> (a Pafivik config, a Ridopel config) of the same width, layers, vocabulary and positions.  The Pafivik layers
    take turns between lightning (heads of 64 keys x 128 values), channel_delta (as many heads of 64 x 128 over half as many
    heads of queries and keys, four taps, inner sizes of 64), attention (heads of 64, a key head for every four, all 64
    dimensions turned) and channel_delta again; each has sixteen experts of the model's width of which a token uses two, and
    a shared expert of the model's width: Ridopel's experts, so that the two differ by their mixers, norms and averages."""
    H = width // 128
    moe = dict(kind="moe", expert=dict(ff=width), router=dict(experts=16, top=2), shared=dict(ff=width))
    delta = dict(type="channel_delta", mlp=moe, mixer=dict(heads=H, kv_heads=max(1, H // 2), dim=64, vdim=128, conv=4, decay_rank=64,
                                                             gate_rank=64))
    kinds = [dict(type="lightning", mlp=moe, mixer=dict(heads=H, dim=64, vdim=128, decay=[1.0 - 2.0 ** -(5 + 3 * h / H) for h in range(H)])),
             delta,
             dict(type="attention", mlp=moe, mixer=dict(heads=width // 64, kv_heads=max(1, width // 256), dim=64, vdim=64, scale=0.125,
                                                        rot=dict(base=10000.0, dims=64))),
             delta]
    paf = dict(architecture="Pafivik", vocab=vocab, width=width, norm=dict(eps=1e-5), embedding=dict(scale=1.0), residual_mult=0.5,
               layers=[kinds[i % 4] for i in range(layers)], max_positions=positions, n_positions=positions, vocab_size=vocab)
    return paf, ridopel_configs(width, layers, vocab, positions)[0]


def dogalorn_configs(width, layers=4, vocab=32000, positions=2048):
    """-> (a Dogalorn config, a Pafivik config) of the same width, layers, vocabulary and positions, both with dense
    feed-forwards four times the width.  The Dogalorn layers: attention in chunks of 512 (heads of 64, a key head for every
    four, a table of 32 distance biases) beside a minGRU of the model's width; Mamba2 (heads of 64 values, twice the width in
    all, states of 128, four taps); Mamba2; the pair again; the stream in two copies; token rows plus rows picked by pairs.
    The Pafivik layers: attention (heads of 64, a key head for every four), lightning (heads of 64 keys x 128 values), lightning,
    attention."""
    H = width // 64
    ff = dict(kind="dense", ff=4 * width)
    par = dict(type="parallel", mlp=ff, mixer=dict(
        left=dict(heads=H, kv_heads=max(1, H // 4), dim=64, vdim=64, scale=0.125, bias_max=400, mask=dict(size=512), bias_buckets=32),
        right=dict(width=width)))
    mam = dict(type="mamba2", mlp=ff, mixer=dict(heads=2 * H, vdim=64, state=128, groups=1, conv=4, norm_groups=1))
    kinds = [par, mam, mam, par]
    dog = dict(architecture="Dogalorn", vocab=vocab, width=width, norm=dict(eps=1e-5), streams=2, logit_scale=1.0,
               embedding=dict(bigram=dict(buckets=100003, mul_prev=7919, mul_cur=4099)), layers=[kinds[i % 4] for i in range(layers)],
               max_positions=positions, n_positions=positions, vocab_size=vocab)
    Hl = width // 128
    att = dict(type="attention", mlp=ff, mixer=dict(heads=H, kv_heads=max(1, H // 4), dim=64, vdim=64, scale=0.125,
                                                    rot=dict(base=10000.0, dims=64)))
    lig = dict(type="lightning", mlp=ff, mixer=dict(heads=Hl, dim=64, vdim=128, decay=[1.0 - 2.0 ** -(5 + 3 * h / Hl) for h in range(Hl)]))
    kinds = [att, lig, lig, att]
    paf = dict(architecture="Pafivik", vocab=vocab, width=width, norm=dict(eps=1e-5), embedding=dict(scale=1.0), residual_mult=0.5,
               layers=[kinds[i % 4] for i in range(layers)], max_positions=positions, n_positions=positions, vocab_size=vocab)
    return dog, paf


def nigilorn_configs(width, layers=4, vocab=32000, positions=2048):
    """-> (a Nigilorn config, a Pafivik config) of the same width, layers, vocabulary and positions.  The Nigilorn layers: a
    selective scan (twice the width in channels, 16 states a channel, a step of rank width / 16, four taps); attention
    (heads of 64, a key head for every four, half of a head turned with a stretched encoding, a window of 256); latent
    attention (heads of 64 + 32, values of 128, a kept key of 224 + 32 numbers, a window of 256); the scan again.  The first
    layer has a dense feed-forward of four times the width, the others sixteen experts of the model's width in four groups
    of which two are kept, two experts a token, and a shared expert of the model's width; a token input of 64 columns a
    layer.  The Pafivik layers (lightning, attention, attention, lightning) have the same feed-forward sizes."""
    H = width // 64
    stretch = dict(factor=4.0, original=512, fast=32.0, slow=1.0)
    ff = dict(kind="dense", ff=4 * width)
    moe = dict(kind="moe", expert=dict(ff=width), router=dict(experts=16, top=2, scale=2.5, groups=dict(count=4, keep=2)), shared=dict(ff=width))
    scan = dict(type="mamba1", mixer=dict(inner=2 * width, state=16, dt_rank=width // 16, conv=4))
    att = dict(type="attention", mixer=dict(heads=H, kv_heads=max(1, H // 4), dim=64, vdim=64, scale=0.125, mask=dict(size=256),
                                            rot=dict(base=10000.0, dims=32, scaling=stretch)))
    lat = dict(type="latent_attention", mixer=dict(heads=width // 128, dim=64, rot_dim=32, vdim=128, kv_rank=224, scale=96 ** -0.5,
                                                   mask=dict(size=256), rot=dict(base=10000.0, dims=32, scaling=stretch)))
    kinds = [dict(scan, mlp=ff), dict(att, mlp=moe), dict(lat, mlp=moe), dict(scan, mlp=moe)]
    nig = dict(architecture="Nigilorn", vocab=vocab, width=width, norm=dict(eps=1e-5), token_side=dict(dim=64),
               layers=[kinds[i % 4] for i in range(layers)], max_positions=positions, n_positions=positions, vocab_size=vocab)
    Hl = width // 128
    pmoe = dict(kind="moe", expert=dict(ff=width), router=dict(experts=16, top=2), shared=dict(ff=width))
    patt = dict(type="attention", mixer=dict(heads=H, kv_heads=max(1, H // 4), dim=64, vdim=64, scale=0.125, rot=dict(base=10000.0, dims=64)))
    lig = dict(type="lightning", mixer=dict(heads=Hl, dim=64, vdim=128, decay=[1.0 - 2.0 ** -(5 + 3 * h / Hl) for h in range(Hl)]))
    kinds = [dict(lig, mlp=ff), dict(patt, mlp=pmoe), dict(patt, mlp=pmoe), dict(lig, mlp=pmoe)]
    paf = dict(architecture="Pafivik", vocab=vocab, width=width, norm=dict(eps=1e-5), embedding=dict(scale=1.0), residual_mult=0.5,
               layers=[kinds[i % 4] for i in range(layers)], max_positions=positions, n_positions=positions, vocab_size=vocab)
    return nig, paf


def fikupel_configs(width, layers=4, vocab=32000, positions=2048):
    """-> (a Fikupel config, a Nigilorn config) of the same width, layers, vocabulary and positions, without Nigilorn's scan and
    token input, so that both have the same kinds of layers in the same order: attention (heads of 64, a key head for every
    four, half of a head turned with a stretched encoding, a window of 256; Fikupel's keeps 16 first tokens) and latent attention
    (heads with values of 128, a kept key of 256 numbers, a window of 256; queries of 64 plain dimensions through a vector of
    half the width, or of 64 + 32 from the stream), again both.  The first layer has a dense feed-forward of four times the width
    (one product up, or a gated one), the others sixteen experts of the model's width of which a token uses two (gated with silu,
    or one product and a squared relu).  Fikupel's stream is four copies."""
    H, Hl = width // 64, width // 128
    ff = dict(kind="dense", ff=4 * width)

    def moe(**router):
        return dict(kind="moe", expert=dict(ff=width), router=dict(experts=16, top=2, **router))

    def att(scaling, **mask):
        return dict(type="attention", mixer=dict(heads=H, kv_heads=max(1, H // 4), dim=64, vdim=64, scale=0.125, mask=dict(size=256, **mask),
                                                 rot=dict(base=10000.0, dims=32, scaling=scaling)))

    def four(a, b, experts):
        kinds = [dict(a, mlp=ff), dict(b, mlp=experts), dict(a, mlp=experts), dict(b, mlp=experts)]
        return dict(vocab=vocab, width=width, norm=dict(eps=1e-5), layers=[kinds[i % 4] for i in range(layers)], max_positions=positions,
                    n_positions=positions, vocab_size=vocab)
    lat = dict(type="latent_attention", mixer=dict(heads=Hl, dim=64, vdim=128, kv_rank=256, q_rank=width // 2, scale=0.125, mask=dict(size=256)))
    fik = dict(four(att(dict(factor=4.0, original=512, low=1.0, high=4.0), keep_first=16), lat, moe()), architecture="Fikupel", streams=4)
    stretch = dict(factor=4.0, original=512, fast=32.0, slow=1.0)
    nlat = dict(type="latent_attention", mixer=dict(heads=Hl, dim=64, rot_dim=32, vdim=128, kv_rank=224, scale=96 ** -0.5, mask=dict(size=256),
                                                    rot=dict(base=10000.0, dims=32, scaling=stretch)))
    nig = dict(four(att(stretch), nlat, moe(scale=2.5, groups=dict(count=4, keep=2))), architecture="Nigilorn")
    return fik, nig


def pepapel_configs(width, layers=4, vocab=32000, positions=2048):
    """-> (a Pepapel config, a Pafivik config) of the same width, vocabulary and positions, with the same mixers and as many
    feed-forwards.  The Pepapel layers: a pair of attention in chunks of 512 (heads of 64, a key head for every four, all dimensions
    turned, four taps) and a delta rule (heads of 64 keys x 128 values, half as many heads of queries and keys, four taps);
    attention over everything (the same heads, a temperature, a soft cap); the pair twice.  The first layer has a dense
    feed-forward of four times the width (gated, with biases), the others sixteen experts of the model's width without a gate, in
    groups with four outputs that return their input, two choices a token.  The Pafivik layers: for every pair an attention layer
    without a feed-forward and a channel_delta layer with one, for every attention an attention layer; dense feed-forwards of
    four times the width, or sixteen gated experts of the model's width of which a token uses two."""
    H, Hd = width // 64, width // 128
    ff = dict(kind="dense", ff=4 * width)
    heads = dict(heads=H, kv_heads=max(1, H // 4), dim=64, vdim=64, scale=0.125)
    delta = dict(heads=Hd, kv_heads=max(1, Hd // 2), dim=64, vdim=128, conv=4)
    moe = dict(kind="moe", expert=dict(ff=width), router=dict(experts=16, identity=4, top=2, groups=dict(count=4, keep=3)))
    pair = dict(type="parallel", mixer=dict(left=dict(heads, conv=4, mask=dict(size=512), rot=dict(base=10000.0, dims=64, scaling=dict(factor=2.0))),
                                            right=delta))
    att = dict(type="attention", mixer=dict(heads, q_temp=dict(coef=0.1, every=256), softcap=30.0))
    kinds = [dict(pair, mlp=dict(ff, limit=7.0)), dict(att, mlp=moe), dict(pair, mlp=moe), dict(pair, mlp=moe)]
    kinds = [kinds[i % 4] for i in range(layers)]
    common = dict(vocab=vocab, width=width, norm=dict(eps=1e-5), embedding=dict(scale=1.0), max_positions=positions, n_positions=positions, vocab_size=vocab)
    pep = dict(common, architecture="Pepapel", postln_alpha=2.5, layers=kinds)
    pmoe = dict(kind="moe", expert=dict(ff=width), router=dict(experts=16, top=2))
    patt = dict(type="attention", mixer=dict(heads, rot=dict(base=10000.0, dims=64)))
    pdelta = dict(type="channel_delta", mixer=dict(delta, decay_rank=64, gate_rank=64))
    others = []
    for layer in kinds:
        mlp = ff if layer["mlp"]["kind"] == "dense" else pmoe
        others += [dict(patt, mlp=None), dict(pdelta, mlp=mlp)] if layer["type"] == "parallel" else [dict(patt, mlp=mlp)]
    return pep, dict(common, architecture="Pafivik", residual_mult=0.5, layers=others)


def pepapel(a):
    """Prefill and decode steps of four Pepapel layers beside seven Pafivik layers with the same mixers and as many feed-forwards
    (the closest of the framework's models: attention with grouped key heads, a delta rule with short convolutions, experts); with
    --kernel-times each model's kernels."""
    return side_by_side(a, ("pepapel", "pafivik"), pepapel_configs)


def fikupel(a):
    """Prefill and decode steps of four Fikupel layers beside four Nigilorn layers of the same kinds and sizes (the closest of the
    framework's models: attention and latent attention in a window, experts); with --kernel-times each model's kernels."""
    return side_by_side(a, ("fikupel", "nigilorn"), fikupel_configs)


def nigilorn(a):
    """Prefill and decode steps of four Nigilorn layers beside four Pafivik layers of the same width and feed-forward sizes
    (the closest of the framework's models: a norm on both sides of every sublayer, an attention over pages, a recurrence
    with a state, experts with a shared one); with --kernel-times each model's kernels."""
    return side_by_side(a, ("nigilorn", "pafivik"), nigilorn_configs)


def dogalorn(a):
    """Prefill and decode steps of four Dogalorn layers beside four Pafivik layers of the same width with the same dense
    feed-forwards (the closest of the framework's models: an attention over pages, recurrences with a matrix state, norms
    without a mean); with --kernel-times each model's kernels."""
    return side_by_side(a, ("dogalorn", "pafivik"), dogalorn_configs)


def pafivik(a):
    """Prefill and decode steps of four Pafivik layers beside four Ridopel layers of the same width (the closest of the
    framework's models: recurrent mixers, an attention, the same experts); with --kernel-times each model's kernels."""
    return side_by_side(a, ("pafivik", "ridopel"), pafivik_configs)


def ridopel(a):
    """Prefill (two prompts of 1,024 tokens in one step) and decode steps (batch 8 and 64 from a context of 512) of four
    Ridopel layers beside four GPT-2 layers of the same width; with --kernel-times each model's kernels, launch by launch."""
    return side_by_side(a, ("ridopel", "gpt2"), ridopel_configs)


def side_by_side(a, names, configs):
    import torch
    from denno_beta_amd.kernels import ops
    out = {}
    for width in ([a.width] if a.width else [1024, 2048]):
        for name, cfg in zip(names, configs(width, a.layers or 4)):
            w = Workloads(a, a.dtype, cfg)
            rec = {"weight_bytes": w.runner.model.weight_bytes(), "cache_bytes_per_token": w.runner.cache.bytes_per_token()}
            w.prefill(1, a.prompts)
            if a.kernel_times:
                ops.time_launches(True)
                w.prefill(1, a.prompts)
                kernel_table(f"{name} width {width}: prefill of {a.prompts} x 1,024 tokens, {a.dtype}")
                for batch in (8, 64):
                    w.decode(batch, 4, 1, blocks=1, on_start=lambda: ops.time_launches(True))
                    kernel_table(f"{name} width {width}: 4 decode steps at batch {batch} from a context of {a.context}, {a.dtype}")
                    ops.time_launches(False)
                ops.time_launches(False)
            else:
                p = w.prefill(3, a.prompts)
                rec["prefill_tok_s"], rec["prefill_ms"] = p["value"], p["ms"]
                for batch in (8, 64):
                    d = w.decode(batch, min(a.steps, 50), a.warmup)
                    rec[f"decode_b{batch}_ms"], rec[f"decode_b{batch}_tok_s"] = d["ms"], d["tok_s"]
            out[f"{name}_{width}"] = rec
            del w
            torch.cuda.empty_cache()
    print(json.dumps(out))


def large_config():
    return baseline_config(3)[0]


def serving(a):
    """GPT-2 Large shape, random weights: 64 requests with prompt lengths uniform in [16, 768], 256
    generated tokens each, greedy, continuous batching with prompt portions of 512.  After the timed
    run four of the requests run again, each alone: their tokens must be the same (32-bit: exactly; in
    bfloat16 a step's kernels depend on its rows, so the count of equal tokens is reported, and the served
    tokens are checked against the 32-bit engine wherever its lead is clear of bfloat16's rounding)."""
    import torch
    from denno_beta_amd.config import EngineOptions
    from denno_beta_amd.engine import Engine, SamplingParams
    cfg = large_config()
    opts = EngineOptions(dtype=a.dtype, page_size=16, cache_tokens=64 * 1024, max_live=64, max_batch_tokens=2048,
                         prefill_chunk=512, use_graphs=not a.no_graphs, seed=0, norms_inside_products=not a.norm_kernels, deferred_sums=not a.no_deferred_sums)
    eng = Engine.from_random(cfg, 0, opts, stored=a.dtype)
    gen = torch.Generator().manual_seed(1)
    lengths = torch.randint(16, 769, (64,), generator=gen).tolist()
    prompts = [torch.randint(0, cfg["vocab_size"], (n,), generator=gen).tolist() for n in lengths]
    sp = SamplingParams(max_tokens=256, temperature=0.0, ignore_eos=True)
    eng.generate(prompts[:2], SamplingParams(max_tokens=4, temperature=0.0, ignore_eos=True))   # warm-up
    eng.records.clear()
    torch.cuda.synchronize()
    t0 = time.perf_counter()
    out = eng.generate(prompts, sp)
    torch.cuda.synchronize()
    dt = time.perf_counter() - t0
    assert all(len(o) == 256 for o in out)
    steps = len(eng.records)
    records = list(eng.records)
    same = []
    for i in (0, 21, 42, 63):
        alone = eng.generate([prompts[i]], sp)[0]
        first_other = next((j for j in range(256) if alone[j] != out[i][j]), 256)
        same.append(first_other)
    if a.dtype == "float32" and min(same) < 256:
        raise SystemExit(f"serving: a request's tokens differ from its run alone (equal tokens before the first "
                         f"difference, of 256: {same})")
    clear_share = None
    if a.dtype == "bfloat16":
        # What can be asked of bfloat16: the 32-bit engine on the same weights, fed each request's prompt and the
        # tokens that were served, says at every generated position which token leads and by how much; where the
        # lead is clear of bfloat16's rounding (twice 0.04 of the row's spread, the bound of the replay tests) the
        # served token must be that one.
        from denno_beta_amd.engine import ModelRunner, StepEntry
        del eng
        r32 = ModelRunner.from_random(cfg, 0, EngineOptions(dtype="float32", page_size=16, cache_tokens=1024, max_live=1,
                                                            use_graphs=False), stored="bfloat16")
        clear = wrong = 0
        for rid, i in enumerate((0, 21, 42, 63)):
            seq = prompts[i] + out[i][:-1]
            r32.start_request(rid)
            logits = r32.step([StepEntry(rid, seq, list(range(len(prompts[i]) - 1, len(seq))))])
            r32.end_request(rid)
            top = logits.topk(2, dim=1)
            sure = (top.values[:, 0] - top.values[:, 1]) > 2 * 0.04 * logits.std(dim=1)
            served = torch.tensor(out[i], device=logits.device)
            clear += int(sure.sum())
            wrong += int((served != top.indices[:, 0])[sure].sum())
        clear_share = clear / (4 * 256)
        if wrong:
            raise SystemExit(f"serving: {wrong} served tokens differ from the 32-bit engine's where its lead is clear "
                             f"({clear} such positions of {4 * 256})")
    print(json.dumps({
        "workload": "GPT-2 Large shape, 64 requests, prompts U[16,768], 256 new tokens, prefill portions of 512",
        "seconds": dt, "generated_tokens": 64 * 256, "generated_tokens_per_s": 64 * 256 / dt,
        "prompt_tokens": sum(lengths), "all_tokens_per_s": (64 * 256 + sum(lengths)) / dt, "steps": steps,
        "mean_rows_per_step": sum(r.rows for r in records) / steps,
        "mixed_steps": sum(1 for r in records if r.decode_rows and r.prefill_rows),
        "preemptions": sum(r.preempted for r in records), "dtype": a.dtype,
        "tokens_equal_to_the_run_alone_before_the_first_difference": same,
        "share_of_positions_where_the_32_bit_lead_is_clear_all_served_as_it_says": clear_share}))


def replay(a):
    """BASELINE.json's configs[4] (GPT-2 Medium shape; --shape xl: configs[2]'s sizes, all 48 layers): random
    weights stored in 32-bit, seeded sequences of 1,024 tokens replayed whole, token by token, in portions of 128 and mixed (four live requests, pages
    used again), every logit compared with the plain implementation's; and the cuttings with each other."""
    import torch
    sys.path.insert(0, os.path.join(ROOT, "tests"))
    import replay_util as U
    from plain.gpt2_plain import PlainGPT2
    from denno_beta_amd.config import EngineOptions
    from denno_beta_amd.engine import ModelRunner
    from denno_beta_amd.engine.replay import TraceReplayer
    from denno_beta_amd.weights import write_model_folder
    import tempfile
    cfg, full = baseline_config({"xl": 2, "large": 3, "medium": 4}[a.shape], a.layers)
    V, n = cfg["vocab_size"], cfg["n_positions"]
    seqs = [torch.randint(0, V, (n,), generator=torch.Generator().manual_seed(100 + i)).tolist()
            for i in range(a.sequences)]
    token_by_token = []
    for base in range(0, len(seqs), 4):          # four requests live at a time, a token of each per step
        group = list(range(base, min(base + 4, len(seqs))))
        for t in range(n):
            token_by_token.append({"step": len(token_by_token), "end": [f"r{i}" for i in group] if t == n - 1 else [],
                                   "entries": [{"id": f"r{i}", "tokens": seqs[i][t:t + 1], "want": [0]} for i in group]})
    traces = {"whole": U.whole_trace(seqs), "token by token": token_by_token,
              "portions of 128": U.chunk_trace(seqs, sizes=(128,)),
              "mixed": U.mixed_trace(seqs, seed=3, sizes=(1, 1, 1, 2, 5, 17, 40, 128))}
    result = {"workload": f"GPT-2 {a.shape} shape, {cfg['n_layer']} of {full} layers, {len(seqs)} sequences of {n} tokens"}
    with tempfile.TemporaryDirectory() as folder:
        print("replay: writing the model and running the plain implementation ...", file=sys.stderr, flush=True)
        write_model_folder(folder, cfg, 4, "float32")
        plain = PlainGPT2.from_folder(folder)
        want = []
        for i, s in enumerate(seqs):
            want.append(plain.logits(s, by_head=True).cuda())
            print(f"replay: plain logits of sequence {i}", file=sys.stderr, flush=True)
        for dtype in ("float32", "bfloat16"):
            whole = None
            for kind, steps in traces.items():
                tokens = U.max_live_tokens(steps)
                runner = ModelRunner.from_folder(folder, EngineOptions(dtype=dtype, page_size=16, cache_tokens=tokens,
                                                                       max_live=4), cast_matrices=True)
                rp = TraceReplayer(runner)
                got = [torch.empty_like(wt) for wt in want]
                pos = {}
                for st in steps:
                    out = rp.run_step(st)
                    k = 0
                    for e in st["entries"]:
                        i, base = int(e["id"][1:]), pos.get(e["id"], 0)
                        m = len(e["want"])
                        got[i][torch.tensor([base + x for x in e["want"]], device="cuda")] = out[k:k + m]
                        k += m
                        pos[e["id"]] = base + len(e["tokens"])
                runner.cache.manager.check()
                worst = max((g - wt).abs().max().item() for g, wt in zip(got, want))
                # the same against what a row's logits differ by among themselves (their standard deviation)
                rel = [(g - wt).abs() / wt.std(dim=1, keepdim=True) for g, wt in zip(got, want)]
                agree = sum((g.argmax(1) == wt.argmax(1)).sum().item() for g, wt in zip(got, want)) / (len(seqs) * n)
                entry = {"worst_difference_from_plain": worst, "greedy_token_agreement": agree,
                         "worst_of_a_rows_spread": max(r.max().item() for r in rel),
                         "mean_of_a_rows_spread": sum(r.mean().item() for r in rel) / len(rel),
                         "steps": len(steps), "pages_used_again": runner.cache.manager.reuse_count(0)}
                if whole is None:
                    whole = got
                else:
                    entry["equal_to_whole_bit_for_bit"] = all(torch.equal(g, wg) for g, wg in zip(got, whole))
                    entry["worst_difference_from_whole"] = max((g - wg).abs().max().item() for g, wg in zip(got, whole))
                result[f"{dtype}, {kind}"] = entry
                print(f"replay: {dtype}, {kind}: {entry}", file=sys.stderr, flush=True)
                del runner, rp
                if kind != "whole":
                    del got
            del whole
    result["largest_logit"] = max(wt.abs().max().item() for wt in want)
    print(json.dumps(result))


if __name__ == "__main__":
    main()
