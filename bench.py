"""Decode and prefill throughput with random bfloat16 weights on one MI355X:
`python bench.py [--gpus 1] [--steps K] [--warmup W]` prints one JSON line.

The headline is the Qwen2.5-7B shape: decoding at batch 8 after 2048-token prompts (`value`, tokens a
second; a step is one decode step of the whole batch through the generation loop: step function,
sampling, host round trip for the stop check), the prompt pass of 2048 tokens (`prefill`), and the decode
step's memory traffic against the HBM peak (`roofline`).  `points` holds decoding at batch 1, 64 and 128,
the same shape at 8192 tokens of context, and the two other workloads of the baseline: the Qwen2.5-1.5B
shape with 32 prompts of unequal lengths sampled at temperature 0.7 (`w15b_*`), and the Qwen2.5-32B shape
with 16 prompts of 512 tokens decoded greedily (`w32b_*`).  `probe` says what this GPU gives a kernel that
only reads memory and one that only feeds the matrix cores; every fraction is given against the published
peak and (`*_of_probe`) against the probe.

The reference measures tokens per second of one chat request including its prompt
(src/main.rs:1123-1143); here decoding is timed alone, the prompt pass is reported beside it, and the
reference's prompt-inclusive figure goes into `end_to_end_tok_per_s`.

`python bench.py --latent` is another measurement with a line of its own (the default workload above is untouched): the
Nikasun design (attention through cached latents with a window, routed experts) at a few sizes that resemble a real
model's layers, beside a Qwen2 shape of the same width, depth, heads and active feed-forward size: prompt pass and
decoding of both, tokens a second.  `python bench.py --masked` does the same for the Sizudra design (attention with normed
heads, mixed values, and in every other layer a score cap, a window that keeps the first positions and a sink; a pair
embedding; norms on the parts' outputs; routed experts without a gate product).  `python bench.py --streams` does it for the Povipel design beside a
Piditar shape of equal size.  `python bench.py --recurrent` does it for the
Piditar design (layers of attention, of a real-gated linear recurrent unit and of a selective state-space mixer, each with a dense
feed-forward).  `python bench.py --matrix-memory` does it for the Rasodra design (a matrix memory, latent attention with a sink and an
element gate, chunked attention whose values are its keys, norms on both sides of every part) beside a Nikasun shape of equal size.
`python bench.py --time-mixing` does it for the Kezasun design (time mixing, windowed attention with a norm over the projection and a gate per head,
experts in groups) beside a Povipel shape of equal size.
"""
import argparse
import gc
import json
import statistics
import sys
import time

PEAK = {"hbm_gbs": 8000.0, "bf16_flops": 2.5e15}     # MI355X: HBM3E 8 TB/s, dense bf16 MFMA 2.5 PFLOP/s


def main():
    ap = argparse.ArgumentParser()
    ap.add_argument("--gpus", type=int, default=1)
    ap.add_argument("--steps", type=int, default=128, help="timed decode steps of the headline")
    ap.add_argument("--warmup", type=int, default=16)
    ap.add_argument("--batch", type=int, default=8)
    ap.add_argument("--prompt-len", type=int, default=2048)
    ap.add_argument("--shape", default="qwen2.5:7b")
    ap.add_argument("--layers", type=int, default=0, help="fewer layers than the shape has (0: all)")
    ap.add_argument("--no-points", action="store_true", help="the headline alone: no other batch sizes, contexts or workloads")
    ap.add_argument("--no-workloads", action="store_true", help="skip the 1.5B and 32B workloads")
    ap.add_argument("--no-long", action="store_true", help="skip the points at 8192 tokens of context")
    ap.add_argument("--no-tune", action="store_true", help="do not let the matrix library try its kernels for the prompt's size")
    ap.add_argument("--no-probe", action="store_true")
    ap.add_argument("--latent", action="store_true", help="measure the Nikasun design beside a Qwen2 shape of equal size instead of the default workload")
    ap.add_argument("--latent-sizes", default="2048,4096", help="widths of the --latent and --masked comparisons")
    ap.add_argument("--masked", action="store_true", help="measure the Sizudra design beside a Qwen2 shape of equal size instead of the default workload")
    ap.add_argument("--recurrent", action="store_true", help="measure the Piditar design beside a Qwen2 shape of equal size instead of the default workload")
    ap.add_argument("--streams", action="store_true", help="measure the Povipel design beside a Piditar shape of equal size instead of the default workload")
    ap.add_argument("--matrix-memory", action="store_true", help="measure the Rasodra design beside a Nikasun shape of equal size instead of the default workload")
    ap.add_argument("--time-mixing", action="store_true", help="measure the Kezasun design beside a Povipel shape of equal size instead of the default workload")
    args = ap.parse_args()
    if args.gpus != 1:
        print("bench.py: this library runs on one GPU; --gpus %d is not supported" % args.gpus)
        return 2

    import torch

    from tq_kv_amd import POLICY, Engine, GenerationParams, Model, generate
    from tq_kv_amd import kernels as K
    from tq_kv_amd.config import catalog

    t_start = time.perf_counter()

    def note(msg):
        print("[bench %.0fs] %s" % (time.perf_counter() - t_start, msg), file=sys.stderr, flush=True)

    # -- what this GPU gives ----------------------------------------------------------------------
    probe = {}
    if not args.no_probe:
        note("probes: a streaming read of 4 GB, a loop of matrix-core products")
        buf = torch.empty(1 << 30, dtype=torch.float32, device="cuda:0")          # 4 GB: far beyond every cache
        buf.fill_(1.0)
        probe["hbm_read_gbs"] = round(K.probe_read(buf), 1)
        del buf
        torch.cuda.empty_cache()
        probe["mfma_bf16_pflops"] = round(K.probe_mfma(), 4)

    def of_probe(value, key):
        return round(value / probe[key], 4) if probe.get(key) else None

    def sizes(raw):
        return dict(L=raw["num_hidden_layers"], H=raw["hidden_size"], I=raw["intermediate_size"], V=raw["vocab_size"],
                    nh=raw["num_attention_heads"], nkv=raw["num_key_value_heads"], d=raw["head_dim"])

    def linear_params(z):
        return z["L"] * (z["H"] * (z["nh"] + 2 * z["nkv"]) * z["d"] + z["nh"] * z["d"] * z["H"] + 3 * z["H"] * z["I"])

    def weight_bytes(z):
        return 2.0 * (linear_params(z) + z["H"] * z["V"])                 # every weight a decode step uses, once

    def kv_bytes_per_token(z):
        return z["L"] * 2 * z["nkv"] * z["d"] * 2.0

    def prefill_flops(z, lens):
        attn = sum(z["L"] * 4.0 * z["nh"] * z["d"] * (n * (n + 1) / 2) for n in lens)
        return 2.0 * sum(lens) * linear_params(z) + attn + 2.0 * z["H"] * z["V"] * len(lens)

    def timed_prefill(engine, prompts, runs):
        """Seconds of the prompt pass of `prompts` (one step, the last place of each wanted), for each of `runs` runs."""
        times = []
        for _ in range(runs):
            slots = [engine.open() for _ in prompts]
            torch.cuda.synchronize()
            t0 = time.perf_counter()
            engine.step([(s, p, [len(p) - 1]) for s, p in zip(slots, prompts)])
            torch.cuda.synchronize()
            times.append(time.perf_counter() - t0)
            for s in slots:
                engine.close(s)
        return times

    def decode(engine, prompts, steps, warmup, params=None):
        """Tokens per second over `steps` decode steps after the prompts, seconds per step, and generated tokens per
        second of the whole run (prompt pass included)."""
        marks, calls = {}, [0]

        def on_tokens(pairs):
            # call i comes when the tokens of draw i are known; draw i+1 needs decode step i+1.  The loop keeps one
            # step under way while it reads a draw, so the device is waited for at the two ends of the timed steps
            # only, and each wait ends just after a step.
            if calls[0] in (warmup, warmup + steps):
                torch.cuda.synchronize()
                marks[calls[0]] = time.perf_counter()
            calls[0] += 1
        params = params or GenerationParams(max_tokens=warmup + steps + 2, temperature=0.0, repeat_penalty=1.0)
        torch.cuda.synchronize()
        t0 = time.perf_counter()
        out = generate(engine, prompts, params, eos_ids=(), on_tokens=on_tokens, max_batch=len(prompts))
        torch.cuda.synchronize()
        whole = time.perf_counter() - t0
        assert all(len(o) == warmup + steps + 2 for o in out)
        seconds = marks[warmup + steps] - marks[warmup]
        return len(prompts) * steps / seconds, seconds / steps, sum(len(o) for o in out) / whole

    def hbm(z, mean_tokens_held, sec_per_step):
        """GB/s of a decode step: the weights once and the cache of the live requests, over its time."""
        return (weight_bytes(z) + mean_tokens_held * kv_bytes_per_token(z)) / sec_per_step / 1e9

    def decode_point(name, z, b_tps, b_sec, mean_tokens_held):
        gbs = hbm(z, mean_tokens_held, b_sec)
        return {name: round(b_tps, 1), name + "_ms": round(b_sec * 1e3, 4), name + "_gbs": round(gbs, 1),
                name + "_frac": round(gbs / PEAK["hbm_gbs"], 4), name + "_frac_of_probe": of_probe(gbs, "hbm_read_gbs")}

    gen = torch.Generator().manual_seed(0)

    def random_prompts(vocab, lens):
        return [torch.randint(0, vocab, (n,), generator=gen).tolist() for n in lens]

    def release():
        gc.collect()
        torch.cuda.empty_cache()

    # -- another design beside the closest existing one -----------------------------------------------
    if args.latent:
        return design_comparison("nikasun", latent_shapes, args, torch, Model, Engine, note, timed_prefill, decode, random_prompts, release)
    if args.masked:
        return design_comparison("sizudra", masked_shapes, args, torch, Model, Engine, note, timed_prefill, decode, random_prompts, release)

    if args.recurrent:
        return design_comparison("piditar", recurrent_shapes, args, torch, Model, Engine, note, timed_prefill, decode, random_prompts, release)
    if args.streams:
        return design_comparison("povipel", streams_shapes, args, torch, Model, Engine, note, timed_prefill, decode, random_prompts, release, beside="piditar")

    if args.matrix_memory:
        return design_comparison("rasodra", memory_shapes, args, torch, Model, Engine, note, timed_prefill, decode, random_prompts, release, beside="nikasun")

    if args.time_mixing:
        return design_comparison("kezasun", mixing_shapes, args, torch, Model, Engine, note, timed_prefill, decode, random_prompts, release, beside="povipel")

    # -- the headline shape -------------------------------------------------------------------------
    raw = dict(catalog.find(args.shape))
    full_layers = raw["num_hidden_layers"]
    if args.layers:
        raw["num_hidden_layers"] = args.layers
    z = sizes(raw)
    ctx_len = raw["max_position_embeddings"]
    long_ctx = 0 if (args.no_points or args.no_long) else 8192
    total_new = args.steps + args.warmup + 2
    if args.prompt_len + total_new > ctx_len:            # other contexts than the shape's own: the position tables grow with them
        ctx_len = (args.prompt_len + total_new + 1023) // 1024 * 1024
    raw["max_position_embeddings"] = max(ctx_len, (long_ctx + 64 + 1023) // 1024 * 1024 if long_ctx else 0)
    note("making random weights for %s (%d layers)" % (args.shape, z["L"]))
    model = Model.random(raw, seed=0, dtype="bfloat16", device="cuda:0")
    per_seq = (args.prompt_len + total_new + 63) // 64 * 64           # positions a sequence holds at the end
    free_bytes = torch.cuda.mem_get_info(0)[0]
    # the other batch sizes, as far as their caches fit beside the weights (long contexts: not all do)
    point_batches = [] if args.no_points else [b for b in (1, 64, 128) if b * per_seq * kv_bytes_per_token(z) < 0.8 * free_bytes]
    room = max([args.batch] + point_batches) * per_seq
    if long_ctx:
        room = max(room, 8 * (long_ctx + 128))
    engine = Engine(model, max_tokens=room)

    def prefill_point(T, runs):
        if not args.no_tune:
            # products of more rows than the own kernels take are the library's: let it try its kernels once for the
            # shapes of the measured prompt pass
            note("library tuning for %d rows" % T)
            model.tune_library(T)
        note("prefill of %d tokens" % T)
        times = timed_prefill(engine, random_prompts(z["V"], [T]), runs + 2)[2:]
        best, median = min(times), statistics.median(times)
        flops = prefill_flops(z, [T])
        return {"value": round(T / median, 1), "tokens": T, "ms": round(median * 1e3, 3), "frac": round(flops / median / PEAK["bf16_flops"], 4),
                "stat": "median of %d runs" % len(times), "ms_best": round(best * 1e3, 3), "value_best": round(T / best, 1),
                "frac_of_probe": of_probe(flops / median / 1e15, "mfma_bf16_pflops")}

    prefill = prefill_point(args.prompt_len, 7)

    note("decode at batch %d" % args.batch)
    tps, sec_per_step, end_to_end = decode(engine, random_prompts(z["V"], [args.prompt_len] * args.batch), args.steps, args.warmup)
    achieved = hbm(z, args.batch * (args.prompt_len + args.warmup + args.steps / 2.0), sec_per_step)
    points = {}
    for batch, steps, warmup in ((1, min(args.steps, 64), 8), (64, min(args.steps, 32), 4), (128, min(args.steps, 16), 4)):
        if batch not in point_batches:
            continue
        note("decode at batch %d" % batch)
        b_tps, b_sec, _ = decode(engine, random_prompts(z["V"], [args.prompt_len] * batch), steps, warmup)
        points.update(decode_point("decode_b%d" % batch, z, b_tps, b_sec, batch * (args.prompt_len + warmup + steps / 2.0)))
    if long_ctx:
        p = prefill_point(long_ctx, 3)
        points.update({"prefill_8k": p["value"], "prefill_8k_ms": p["ms"], "prefill_8k_frac": p["frac"], "prefill_8k_frac_of_probe": p["frac_of_probe"]})
        note("decode at batch 8 after prompts of %d tokens" % long_ctx)
        b_tps, b_sec, _ = decode(engine, random_prompts(z["V"], [long_ctx] * 8), 32, 4)
        points.update(decode_point("decode_b8_8k", z, b_tps, b_sec, 8 * (long_ctx + 4 + 16.0)))
    packed = bool(POLICY["packed"])
    engine = model = None
    release()

    # -- the baseline's other workloads ---------------------------------------------------------------
    workloads = {}
    if not (args.no_points or args.no_workloads):
        # Qwen2.5-1.5B shape: 32 prompts of unequal lengths (uniform in 16..1024), 128 decode steps at temperature 0.7
        raw15 = dict(catalog.find("qwen2.5:1.5b"))
        z15 = sizes(raw15)
        note("making random weights for qwen2.5:1.5b")
        model = Model.random(raw15, seed=0, dtype="bfloat16", device="cuda:0")
        lens = torch.randint(16, 1025, (32,), generator=torch.Generator().manual_seed(1)).tolist()
        engine = Engine(model, max_tokens=sum((n + 128 + 16 + 2 + 63) // 64 * 64 for n in lens))
        prompts = random_prompts(z15["V"], lens)

        def sampled(n):
            return GenerationParams(max_tokens=n, temperature=0.7, top_k=0, top_p=1.0, repeat_penalty=1.0, seed=0)
        if not args.no_tune:
            model.tune_library(sum(lens))
        decode(engine, prompts[:2], 2, 1, sampled(5))                  # untimed: the sampler's first calls
        note("1.5B shape: 32 prompts of %d..%d tokens, 128 steps at temperature 0.7" % (min(lens), max(lens)))
        first = statistics.median(timed_prefill(engine, prompts, 4)[1:])
        w_tps, w_sec, w_e2e = decode(engine, prompts, 128, 16, sampled(128 + 16 + 2))
        points.update(decode_point("w15b_decode", z15, w_tps, w_sec, sum(lens) + 32 * (16 + 64.0)))
        points.update({"w15b_prefill": round(sum(lens) / first, 1), "w15b_prefill_ms": round(first * 1e3, 3),
                       "w15b_prefill_frac": round(prefill_flops(z15, lens) / first / PEAK["bf16_flops"], 4), "w15b_end_to_end": round(w_e2e, 1)})
        workloads["w15b"] = {"model": "qwen2.5:1.5b", "layers": z15["L"], "hidden": z15["H"], "heads": z15["nh"], "kv_heads": z15["nkv"],
                             "head_dim": z15["d"], "intermediate": z15["I"], "vocab": z15["V"], "batch": 32,
                             "prompt_lens": "uniform in 16..1024 (seed 1), %d tokens in all" % sum(lens), "steps": 128, "warmup": 16,
                             "sampling": "temperature 0.7 (no top-k, no top-p, no repeat penalty)", "seq_len": raw15["max_position_embeddings"]}
        engine = model = None
        release()

        # Qwen2.5-32B shape: 16 prompts of 512 tokens, 256 greedy decode steps
        raw32 = dict(catalog.find("qwen2.5:32b"))
        z32 = sizes(raw32)
        note("making random weights for qwen2.5:32b (%.0f GB, and their packed copy)" % (weight_bytes(z32) / 1e9))
        model = Model.random(raw32, seed=0, dtype="bfloat16", device="cuda:0")
        engine = Engine(model, max_tokens=16 * ((512 + 256 + 8 + 2 + 63) // 64 * 64))
        prompts = random_prompts(z32["V"], [512] * 16)
        if not args.no_tune:
            model.tune_library(16 * 512)
        note("32B shape: 16 prompts of 512 tokens, 256 greedy steps")
        first = statistics.median(timed_prefill(engine, prompts, 4)[1:])
        w_tps, w_sec, w_e2e = decode(engine, prompts, 256, 8)
        points.update(decode_point("w32b_decode", z32, w_tps, w_sec, 16 * (512 + 8 + 128.0)))
        points.update({"w32b_prefill": round(16 * 512 / first, 1), "w32b_prefill_ms": round(first * 1e3, 3),
                       "w32b_prefill_frac": round(prefill_flops(z32, [512] * 16) / first / PEAK["bf16_flops"], 4), "w32b_end_to_end": round(w_e2e, 1)})
        workloads["w32b"] = {"model": "qwen2.5:32b", "layers": z32["L"], "hidden": z32["H"], "heads": z32["nh"], "kv_heads": z32["nkv"],
                             "head_dim": z32["d"], "intermediate": z32["I"], "vocab": z32["V"], "batch": 16, "prompt_len": 512,
                             "steps": 256, "warmup": 8, "sampling": "greedy", "seq_len": raw32["max_position_embeddings"]}
        engine = model = None
        release()
    note("done")
    line = {
        "metric": "decode tok/s @ batch %d, %s shape" % (args.batch, args.shape), "value": round(tps, 1), "unit": "tokens/s",
        "n_gpus": 1, "steps": args.steps, "warmup": args.warmup, "ms_per_step": round(sec_per_step * 1e3, 4),
        "higher_is_better": True, "scaling": "weak", "vs_baseline": None, "dtype": "bf16", "data": "synthetic",
        "config": {"model": args.shape, "global_batch": args.batch, "seq_len": ctx_len, "parallelism": "single-gpu",
                   "layers": z["L"], "layers_of_shape": full_layers, "hidden": z["H"], "heads": z["nh"], "kv_heads": z["nkv"],
                   "head_dim": z["d"], "intermediate": z["I"], "vocab": z["V"], "prompt_len": args.prompt_len,
                   "new_tokens": total_new, "weights": "random N(0,0.02)", "sampling": "greedy",
                   "library_tuning": not args.no_tune, "packed_weight_copy": packed, "position_table": raw["max_position_embeddings"]},
        "prefill": prefill,
        "roofline": {"bound": "hbm", "achieved": round(achieved, 1), "peak": PEAK["hbm_gbs"], "unit": "GB/s",
                     "frac": round(achieved / PEAK["hbm_gbs"], 4), "frac_of_probe": of_probe(achieved, "hbm_read_gbs")},
        "probe": probe,
        "points": points,
        "workloads": workloads,
        # the reference's figure: generated tokens over the whole run, prompt pass included (src/main.rs:1139-1143)
        "end_to_end_tok_per_s": round(end_to_end, 1),
    }
    print(json.dumps(line))
    return 0


def latent_shapes(width, layers=4):
    """A Nikasun configuration and a Qwen2 one of the same width, depth, heads, head size and active feed-forward size."""
    heads, dim = width // 128, 128
    experts, top, ff = (32, 4, width // 2) if width <= 2048 else (64, 6, width // 4)
    shared = 2 * ff
    active = top * ff + shared
    mixer = {"heads": heads, "dim": dim, "rot_dim": 64, "vdim": dim, "q_rank": 3 * width // 8, "kv_rank": 512, "scale": (dim + 64) ** -0.5,
             "rot": {"base": 10000.0, "dims": 64}, "mask": {"size": 1024}}
    moe = {"kind": "moe", "router": {"experts": experts, "top": top, "scale": 1.0}, "expert": {"ff": ff, "limit": 7.0},
           "shared": {"ff": shared, "limit": 7.0}}
    lay = []
    for l in range(layers):
        m = dict(mixer)
        if l % 2 == 1:
            m["kv_from"] = l - 1
        lay.append({"type": "latent_attention", "mixer": m, "mlp": {"kind": "dense", "ff": active} if l == 0 else moe})
    nikasun = {"architecture": "Nikasun", "vocab": 32000, "width": width, "embedding": {"scale": width ** 0.5}, "norm": {"eps": 1e-5},
               "layers": lay, "max_positions": 8192}
    qwen2 = {"architectures": ["Qwen2ForCausalLM"], "model_type": "qwen2", "hidden_act": "silu", "vocab_size": 32000, "hidden_size": width,
             "intermediate_size": active, "num_hidden_layers": layers, "num_attention_heads": heads, "num_key_value_heads": max(1, heads // 4),
             "head_dim": dim, "rms_norm_eps": 1e-5, "rope_theta": 10000.0, "max_position_embeddings": 8192, "tie_word_embeddings": True,
             "use_sliding_window": True, "sliding_window": 1024, "max_window_layers": 0}
    return nikasun, qwen2, {"width": width, "layers": layers, "heads": heads, "experts": experts, "top": top, "expert_ff": ff,
                            "shared_ff": shared, "active_ff": active, "q_rank": mixer["q_rank"], "kv_rank": 512, "window": 1024}


def masked_shapes(width, layers=4):
    """A Sizudra configuration and a Qwen2 one of the same width, depth, heads, head size and active feed-forward products."""
    heads, dim = width // 128, 128
    kv_heads = max(1, heads // 4)
    experts, top, ff = (32, 4, width // 2) if width <= 2048 else (64, 6, width // 4)
    shared = 2 * ff
    # an expert is two products, a gated feed-forward three: the dense size whose three products equal the active experts' two
    active = 2 * (top * ff + shared) // 3 // 256 * 256
    plain = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": dim ** -0.5, "rot": {"base": 10000.0, "dims": 64}, "v_mix": True}
    second = dict(plain, softcap=30.0, mask={"size": 1024, "keep_first": 4})
    moe = {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff}, "shared": {"ff": shared}}
    lay = [{"type": "attention_2" if l % 2 else "attention", "mixer": second if l % 2 else plain,
            "mlp": {"kind": "dense", "ff": active} if l == 0 else moe} for l in range(layers)]
    sizudra = {"architecture": "Sizudra", "vocab": 32000, "width": width, "embedding": {"bigram": {"buckets": 65521, "mul_prev": 31, "mul_cur": 17}},
               "norm": {"eps": 1e-5}, "layers": lay, "max_positions": 8192}
    qwen2 = {"architectures": ["Qwen2ForCausalLM"], "model_type": "qwen2", "hidden_act": "silu", "vocab_size": 32000, "hidden_size": width,
             "intermediate_size": active, "num_hidden_layers": layers, "num_attention_heads": heads, "num_key_value_heads": kv_heads,
             "head_dim": dim, "rms_norm_eps": 1e-5, "rope_theta": 10000.0, "max_position_embeddings": 8192, "tie_word_embeddings": False,
             "use_sliding_window": True, "sliding_window": 1024, "max_window_layers": layers // 2}
    return sizudra, qwen2, {"width": width, "layers": layers, "heads": heads, "kv_heads": kv_heads, "experts": experts, "top": top, "expert_ff": ff,
                            "shared_ff": shared, "dense_ff": active, "window": 1024, "keep_first": 4}


def recurrent_shapes(width, layers=4):
    """A Piditar configuration (attention, recurrent unit, state-space mixer, recurrent unit) and a Qwen2 one of the same width, depth, heads,
    head size and feed-forward size."""
    heads, dim = width // 128, 128
    kv_heads = max(1, heads // 4)
    ff = 3 * width
    attention = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": dim ** -0.5, "softcap": 50.0, "rot": {"base": 10000.0, "dims": 64}}
    rglru = {"width": width, "blocks": heads, "conv": 4}
    mamba2 = {"heads": 2 * width // 64, "vdim": 64, "state": 128, "groups": 1, "conv": 4, "norm_groups": 1}
    kinds = [("attention", attention), ("rglru", rglru), ("mamba2", mamba2), ("rglru", rglru)]
    lay = [{"type": kinds[l % 4][0], "mixer": kinds[l % 4][1], "mlp": {"kind": "dense", "ff": ff}} for l in range(layers)]
    piditar = {"architecture": "Piditar", "vocab": 32000, "width": width, "embedding": {"scale": width ** 0.5}, "norm": {"eps": 1e-5}, "layers": lay,
               "loop": {"start": 0, "stop": layers, "times": 1}, "max_positions": 8192}
    qwen2 = {"architectures": ["Qwen2ForCausalLM"], "model_type": "qwen2", "hidden_act": "silu", "vocab_size": 32000, "hidden_size": width,
             "intermediate_size": ff, "num_hidden_layers": layers, "num_attention_heads": heads, "num_key_value_heads": kv_heads,
             "head_dim": dim, "rms_norm_eps": 1e-5, "rope_theta": 10000.0, "max_position_embeddings": 8192, "tie_word_embeddings": True}
    return piditar, qwen2, {"width": width, "layers": layers, "heads": heads, "kv_heads": kv_heads, "ff": ff, "rglru_width": width, "rglru_blocks": heads,
                            "mamba2_heads": mamba2["heads"], "mamba2_state": 128, "conv": 4}


def streams_shapes(width, layers=4):
    """A Povipel configuration (the stream in four copies; attention over a window plus pooled blocks beside a gated linear attention, and
    retention, in turn; a dense feed-forward and routed experts in turn) and a Piditar one (attention, recurrent unit, state-space mixer,
    recurrent unit; gated dense feed-forwards) of the same width, depth, attention heads and head size, and as many multiply-adds in the
    active feed-forward products."""
    piditar, _, base = recurrent_shapes(width, layers)
    heads, dim, kv_heads = base["heads"], 128, base["kv_heads"]
    left = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": dim ** -0.5, "mask": {"size": 1024, "pool": 16}, "rot": {"base": 10000.0, "dims": 64}}
    right = {"heads": width // 256, "dim": 128, "vdim": 256, "tau": 16.0}
    retention = {"heads": width // 128, "dim": 128, "vdim": 256, "rot": {"base": 10000.0, "dims": 128},
                 "decay": [1.0 - 2.0 ** (-5.0 - 3.0 * h / max(1, width // 128 - 1)) for h in range(width // 128)]}
    # a gated feed-forward of 3 W holds 9 W^2 weights: the same in two products, and in the three products of each of 4 chosen experts
    dense = {"kind": "dense", "ff": 9 * width // 2}
    moe = {"kind": "moe", "expert": {"ff": 3 * width // 4}, "router": {"experts": 32, "top": 4}}
    kinds = [("parallel", {"left": left, "right": right}, dense), ("retention", retention, moe), ("parallel", {"left": left, "right": right}, moe),
             ("retention", retention, dense)]
    lay = [{"type": kinds[l % 4][0], "mixer": kinds[l % 4][1], "mlp": kinds[l % 4][2]} for l in range(layers)]
    povipel = {"architecture": "Povipel", "vocab": 32000, "width": width, "embedding": {"scale": width ** 0.5}, "norm": {"eps": 1e-5}, "streams": 4,
               "logit_softcap": 30.0, "layers": lay, "loop": {"start": 0, "stop": layers, "times": 1}, "max_positions": 8192}
    return povipel, piditar, {"width": width, "layers": layers, "heads": heads, "kv_heads": kv_heads, "streams": 4, "window": 1024, "pool": 16,
                              "linear_heads": right["heads"], "linear_dim": 128, "linear_vdim": 256, "retention_heads": retention["heads"],
                              "dense_ff": dense["ff"], "experts": 32, "top": 4, "expert_ff": moe["expert"]["ff"], "beside_ff": base["ff"]}


def memory_shapes(width, layers=4):
    """A Rasodra configuration (matrix memory without a feed-forward, latent attention, chunked attention, latent attention) and a Nikasun one (latent
    attention in every layer, the first without a feed-forward) of the same width, depth, heads, head sizes and latent, and as many
    multiply-adds in the feed-forward products."""
    heads, dim = width // 128, 128
    kv_heads = max(1, heads // 4)
    ff = 4 * width
    rot = {"base": 10000.0, "dims": 64}
    memory = {"heads": width // 256, "dim": 128, "vdim": 256, "gate_cap": 15.0}
    latent = {"heads": heads, "dim": dim, "rot_dim": 64, "vdim": dim, "kv_rank": 512, "scale": (dim + 64) ** -0.5, "rot": rot}
    chunked = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": dim ** -0.5, "mask": {"size": 1024}, "rot": rot}
    dense = {"kind": "dense", "ff": ff}
    kinds = [("mlstm", memory, None), ("latent_attention", latent, dense), ("attention", chunked, dense), ("latent_attention", latent, dense)]
    lay = [{"type": kinds[l % 4][0], "mixer": kinds[l % 4][1], "mlp": kinds[l % 4][2]} for l in range(layers)]
    rasodra = {"architecture": "Rasodra", "vocab": 32000, "width": width, "norm": {"eps": 1e-5}, "layers": lay, "max_positions": 8192}
    # a gated feed-forward is three products, Rasodra's two
    gated = {"kind": "dense", "ff": 2 * ff // 3 // 256 * 256}
    other = dict(latent, q_rank=3 * width // 8, mask={"size": 8192})
    nikasun = {"architecture": "Nikasun", "vocab": 32000, "width": width, "embedding": {"scale": width ** 0.5}, "norm": {"eps": 1e-5}, "max_positions": 8192,
               "layers": [{"type": "latent_attention", "mixer": other, "mlp": gated if l % 4 else None} for l in range(layers)]}
    return rasodra, nikasun, {"width": width, "layers": layers, "memory_heads": memory["heads"], "memory_dim": 128, "memory_vdim": 256, "heads": heads,
                              "kv_heads": kv_heads, "head_dim": dim, "kv_rank": 512, "rot_dim": 64, "chunk": 1024, "ff": ff, "beside_ff": gated["ff"],
                              "beside_q_rank": other["q_rank"]}


def mixing_shapes(width, layers=4):
    """A Kezasun configuration (attention, time mixing, attention on the first one's keys and values, time mixing; experts in every layer) and a
    Povipel one of one copy of the stream (attention over a window and pooled blocks beside a gated linear attention, and retention, in turn;
    experts in every layer) of the same width, depth, heads and experts."""
    heads, dim = width // 128, 128
    kv_heads = max(1, heads // 4)
    rot = {"base": 10000.0, "dims": 64}
    mixing = {"heads": width // 64, "dim": 64}
    attention = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": dim ** -0.5, "mask": {"size": 1024},
                 "rot": dict(rot, scaling={"factor": 8.0, "low": 1.0, "high": 4.0, "original": 8192})}
    moe = {"kind": "moe", "expert": {"ff": 3 * width // 4}, "router": {"experts": 30, "top": 4, "identity": 2, "groups": {"count": 4, "keep": 2}}}
    kinds = [("attention", attention), ("wkv", mixing), ("attention", dict(attention, kv_from=0)), ("wkv", mixing)]
    lay = [{"type": kinds[l % 4][0], "mixer": kinds[l % 4][1], "mlp": moe} for l in range(layers)]
    kezasun = {"architecture": "Kezasun", "vocab": 32000, "width": width, "norm": {"eps": 1e-5}, "residual_mult": 0.7, "layers": lay, "max_positions": 8192}
    left = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": dim ** -0.5, "mask": {"size": 1024, "pool": 16}, "rot": rot}
    right = {"heads": width // 256, "dim": 128, "vdim": 256, "tau": 16.0}
    retention = {"heads": width // 64, "dim": 64, "vdim": 64, "rot": {"base": 10000.0, "dims": 64},
                 "decay": [1.0 - 2.0 ** (-5.0 - 3.0 * h / max(1, width // 64 - 1)) for h in range(width // 64)]}
    other = {"kind": "moe", "expert": {"ff": 3 * width // 4}, "router": {"experts": 32, "top": 4}}
    kinds = [("parallel", {"left": left, "right": right}), ("retention", retention)]
    povipel = {"architecture": "Povipel", "vocab": 32000, "width": width, "embedding": {"scale": width ** 0.5}, "norm": {"eps": 1e-5}, "max_positions": 8192,
               "layers": [{"type": kinds[l % 2][0], "mixer": kinds[l % 2][1], "mlp": other} for l in range(layers)]}
    return kezasun, povipel, {"width": width, "layers": layers, "mixing_heads": mixing["heads"], "mixing_dim": 64, "heads": heads, "kv_heads": kv_heads, "head_dim": dim,
                              "window": 1024, "experts": 30, "identity_experts": 2, "top": 4, "groups": 4, "groups_kept": 2, "expert_ff": moe["expert"]["ff"],
                              "beside_linear_heads": right["heads"], "beside_linear_dim": 128, "beside_linear_vdim": 256, "beside_retention_heads": retention["heads"]}


def design_comparison(design, shapes, args, torch, Model, Engine, note, timed_prefill, decode, random_prompts, release, beside="qwen2"):
    prompt_len, out = 2048, {}
    for width in [int(x) for x in args.latent_sizes.split(",")]:
        other, qwen2, sizes = shapes(width)
        row = {"sizes": sizes}
        for name, raw in ((design, other), (beside, qwen2)):
            note("width %d, %s: random weights" % (width, name))
            model = Model.random(raw, seed=0, dtype="bfloat16", device="cuda:0")
            engine = Engine(model, max_tokens=64 * (prompt_len + 256))
            if not args.no_tune:
                model.tune_library(prompt_len)
            times = timed_prefill(engine, random_prompts(32000, [prompt_len]), 5)[2:]
            row[name + "_prefill_tok_s"] = round(prompt_len / statistics.median(times), 1)
            row[name + "_prefill_ms"] = round(statistics.median(times) * 1e3, 3)
            for batch in (8, 64):
                note("width %d, %s: decode at batch %d" % (width, name, batch))
                tps, sec, _ = decode(engine, random_prompts(32000, [prompt_len] * batch), min(args.steps, 32), 4)
                row["%s_decode_b%d_tok_s" % (name, batch)] = round(tps, 1)
                row["%s_decode_b%d_ms" % (name, batch)] = round(sec * 1e3, 4)
            engine = model = None
            release()
        for key in ("prefill_tok_s", "decode_b8_tok_s", "decode_b64_tok_s"):
            row["ratio_" + key] = round(row[design + "_" + key] / row[beside + "_" + key], 3)
        out["width_%d" % width] = row
    first = out["width_%d" % int(args.latent_sizes.split(",")[0])]
    print(json.dumps({"metric": "decode tok/s @ batch 8, %s design at width %s" % (design.capitalize(), args.latent_sizes.split(",")[0]),
                      "value": first[design + "_decode_b8_tok_s"], "unit": "tokens/s", "n_gpus": 1, "steps": min(args.steps, 32), "warmup": 4,
                      "ms_per_step": first[design + "_decode_b8_ms"], "higher_is_better": True, "scaling": "weak", "vs_baseline": None,
                      "dtype": "bf16", "data": "synthetic", "config": {"model": design + " beside " + beside + " at equal size", "prompt_len": prompt_len,
                                                                     "weights": "random"}, "comparison": out}))
    return 0


if __name__ == "__main__":
    sys.exit(main())
