"""Decode and prefill throughput of the engine on one MI355X.

    python bench.py [--gpus 1] [--steps K] [--warmup W] [--model qwen3-4b|qwen3-8b|qwen3-14b|qwen3-32b|qwen3-0.6b|qwen3-1.7b]

The default run has the layer sizes of Qwen3-4B with random weights (bfloat16),
eight requests decoding from 1,024-token random prompts in a cache pool sized
for the benchmark context, and prints ONE JSON line: decoded tokens a second
at batch 8 (``value``), the same at batch 1 and 64 (``points``), the prefill of
one 2,048-token prompt, and the decode step's memory roofline.  A "step" is one
decode step: every request's last token through the model, and the next token
sampled (greedy) and read back.  The sampled tokens are fed to the next step on
the device and read by the host while that step runs (``--no-overlap`` reads
them before the next step is launched).  Everything goes through the engine's
own step function, cache and kernels.

Protocol (after tools/validate_l4.py:136-183 of the reference): W untimed steps,
then K steps each bracketed by a pair of device events; the line reports their
minimum, 10th percentile, median, 90th percentile and maximum, ``value`` is
batch / median, and ``ms_per_step_wall`` is the host's clock over the same K
steps (synchronised on both sides).  The roofline is given against the
published peak and against a streaming read measured when the program starts.

``--through scheduler`` decodes through ``ConcurrentGenerationEngine.step()``
(admission, selection, sampling and finishing included) instead of calling the
step function directly.  ``--workload mixed`` runs requests with prompts of
random lengths to completion through the scheduler and reports the whole job.
``--phase check`` times nothing: it feeds one prompt of ``--prefill-tokens`` whole
and eight more tokens one by one through the chosen model in bfloat16 and in
32-bit, built from the same seed, and prints how far the logits lie apart.
"""

from __future__ import annotations

import argparse
import json
import sys
import time
from pathlib import Path

ROOT = Path(__file__).resolve().parent
sys.path.insert(0, str(ROOT))

# MI355X published peaks
HBM_BYTES_PER_S = 8.0e12
PEAK_FLOPS = {"bf16": 2.5e15, "fp32": 157.3e12}


def _qwen3(**sizes) -> dict:
    base = {"architectures": ["Qwen3ForCausalLM"], "model_type": "qwen3", "hidden_act": "silu",
            "vocab_size": 151936, "num_key_value_heads": 8, "head_dim": 128, "max_position_embeddings": 262144,
            "rms_norm_eps": 1e-6, "attention_bias": False, "eos_token_id": 151645}
    base.update(sizes)
    return base


# Sizes and workloads of the three models the benchmark names (and one between them); the first is the default.
MODELS = {
    "qwen3-4b": {
        "label": "Qwen3-4B",
        "config": _qwen3(hidden_size=2560, intermediate_size=9728, num_hidden_layers=36, num_attention_heads=32,
                         rope_theta=5000000.0, tie_word_embeddings=True),
        "batch": 8, "points": "1,64", "prompt_len": 1024, "context": 8192,
    },
    "qwen3-8b": {
        "label": "Qwen3-8B",
        "config": _qwen3(hidden_size=4096, intermediate_size=12288, num_hidden_layers=36, num_attention_heads=32,
                         rope_theta=1000000.0, tie_word_embeddings=False),
        "batch": 8, "points": "1,64", "prompt_len": 1024, "context": 8192,
    },
    # beside the three: the sizes between them, so that choices measured at those are checked at one more width
    "qwen3-14b": {
        "label": "Qwen3-14B",
        "config": _qwen3(hidden_size=5120, intermediate_size=17408, num_hidden_layers=40, num_attention_heads=40,
                         rope_theta=1000000.0, tie_word_embeddings=False),
        "batch": 8, "points": "1,64", "prompt_len": 1024, "context": 8192,
    },
    # ... and the two smallest of the family, whose products have fewer blocks than the chip has CUs
    "qwen3-0.6b": {
        "label": "Qwen3-0.6B",
        "config": _qwen3(hidden_size=1024, intermediate_size=3072, num_hidden_layers=28, num_attention_heads=16,
                         rope_theta=1000000.0, tie_word_embeddings=True),
        "batch": 8, "points": "1,64", "prompt_len": 1024, "context": 8192,
    },
    "qwen3-1.7b": {
        "label": "Qwen3-1.7B",
        "config": _qwen3(hidden_size=2048, intermediate_size=6144, num_hidden_layers=28, num_attention_heads=16,
                         rope_theta=1000000.0, tie_word_embeddings=True),
        "batch": 8, "points": "1,64", "prompt_len": 1024, "context": 8192,
    },
    "qwen3-32b": {
        "label": "Qwen3-32B",
        "config": _qwen3(hidden_size=5120, intermediate_size=25600, num_hidden_layers=64, num_attention_heads=64,
                         rope_theta=1000000.0, tie_word_embeddings=False),
        "batch": 8, "points": "1,32", "prompt_len": 2048, "context": 16384,
    },
}


def parse_args():
    parser = argparse.ArgumentParser()
    parser.add_argument("--gpus", type=int, default=1)
    parser.add_argument("--steps", type=int, default=50)
    parser.add_argument("--warmup", type=int, default=10)
    parser.add_argument("--model", choices=sorted(MODELS), default="qwen3-4b")
    parser.add_argument("--batch", type=int, default=None)
    parser.add_argument("--prompt-len", type=int, default=None)
    parser.add_argument("--context", type=int, default=None)
    parser.add_argument("--prefill-tokens", type=int, default=2048)
    parser.add_argument("--block-size", type=int, default=16)
    parser.add_argument("--layers", type=int, default=None, help="run fewer layers than the model has")
    parser.add_argument("--dtype", choices=("bf16", "fp32"), default="bf16")
    parser.add_argument("--points", default=None, help="other decode batch sizes to report")
    parser.add_argument("--widths", default="1024,2048,4096",
                        help="--phase design: model widths at which Mazanex and Qwen3 are measured side by side")
    parser.add_argument("--design", choices=("mazanex", "rekezen", "malusun", "dubizen", "talapel", "budanex"), default="mazanex",
                        help="--phase design: which design is measured beside Qwen3")
    parser.add_argument("--only", default="", help="--phase design: measure this model of the comparison alone")
    parser.add_argument("--phase", choices=("all", "decode", "prefill", "micro", "check", "design"), default="all",
                        help="run one phase only (for profiles); the record then holds that phase alone")
    parser.add_argument("--through", choices=("step", "scheduler"), default="step",
                        help="decode by calling the step function, or through the scheduler's step()")
    parser.add_argument("--workload", choices=("steady", "mixed"), default="steady",
                        help="mixed: requests with prompts of random lengths run to completion through the scheduler")
    parser.add_argument("--requests", type=int, default=64, help="mixed workload: number of requests")
    parser.add_argument("--prompt-range", default="128,4096", help="mixed workload: prompt lengths, uniform")
    parser.add_argument("--new-tokens", type=int, default=256, help="mixed workload: tokens generated per request")
    parser.add_argument("--token-budget", type=int, default=2048, help="scheduler: tokens a step")
    parser.add_argument("--sampled", action="store_true",
                        help="through the scheduler: draw with temperature 0.8, top-k 50, top-p 0.9 instead of the arg-max")
    parser.add_argument("--no-overlap", dest="overlap", action="store_false",
                        help="read every step's tokens back before the next step is launched")
    parser.add_argument("--seed", type=int, default=0)
    args = parser.parse_args()
    chosen = MODELS[args.model]
    for name in ("batch", "prompt_len", "context", "points"):
        if getattr(args, name) is None:
            setattr(args, name, chosen[name])
    return args


def weight_bytes(model) -> int:
    """Bytes of every tensor a decode step reads once (the embedding matrix
    counts once: as the head of a tied model, or as the head's own matrix)."""
    seen, total = set(), 0

    def walk(value, depth=0):
        nonlocal total
        if hasattr(value, "data_ptr") and hasattr(value, "element_size"):
            if value.data_ptr() not in seen:
                seen.add(value.data_ptr())
                total += value.numel() * value.element_size()
        elif isinstance(value, dict) and depth < 6:          # tensors by name, parts by name (mixers side by side)
            for inner in value.values():
                walk(inner, depth + 1)
        elif hasattr(value, "param_specs") and hasattr(value, "ctx") and depth < 6 and id(value) not in seen:
            seen.add(id(value))
            for inner in vars(value).values():
                walk(inner, depth + 1)

    for part in model.parts():
        walk(part)
    if not getattr(model.head, "tied", False):
        total -= model.embedding.weight.numel() * model.embedding.weight.element_size()
    return total


def percentile(ordered: list[float], fraction: float) -> float:
    """Linear interpolation between the two nearest of the sorted values."""
    at = fraction * (len(ordered) - 1)
    low = int(at)
    high = min(low + 1, len(ordered) - 1)
    return ordered[low] + (ordered[high] - ordered[low]) * (at - low)


def spread(times_ms: list[float]) -> dict:
    ordered = sorted(times_ms)
    return {"min": round(ordered[0], 4), "p10": round(percentile(ordered, 0.1), 4),
            "median": round(percentile(ordered, 0.5), 4), "p90": round(percentile(ordered, 0.9), 4),
            "max": round(ordered[-1], 4)}


def micro_benchmarks() -> int:
    """The three kernel measurements that the reference publishes (docs/benchmarks.md:27-29,
    results/l4-v0.1.0.json:51-65; one NVIDIA L4), with its shapes and its protocol
    (tools/validate_l4.py:136-183: 10 warm-up calls, 50 timed ones, a pair of device events around
    each call, the median), on this engine's kernels.  A call is timed as the reference times it,
    from the host, so a few microseconds of every figure are the launch."""
    import torch

    from forge_engine_amd.kernels import ops

    device = torch.device("cuda:0")
    generator = torch.Generator(device=device).manual_seed(0)

    def rand(*shape, dtype=torch.bfloat16):
        return torch.randn(*shape, generator=generator, device=device, dtype=torch.float32).to(dtype)

    def measure(fn):
        for _ in range(10):
            fn()
        torch.cuda.synchronize()
        events = [(torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)) for _ in range(50)]
        for begin, end in events:
            begin.record()
            fn()
            end.record()
        torch.cuda.synchronize()
        return spread([begin.elapsed_time(end) for begin, end in events])

    record = {"phase": "micro", "protocol": "10 warm-up, 50 timed, device events around each call, milliseconds"}

    # residual add + RMSNorm, [512, 2560]: the stream is float32 here, the update and the result bfloat16
    stream, update = rand(512, 2560, dtype=torch.float32), rand(512, 2560)
    weight, normed = rand(2560, dtype=torch.float32), torch.empty(512, 2560, dtype=torch.bfloat16, device=device)
    record["residual_add_rms_norm_512x2560"] = dict(measure(lambda: ops.add_rmsnorm(stream, update, weight, 1e-6, normed)),
                                                    reference_l4_ms=0.0850)

    def paged(context, q_tokens, q_heads, kv_heads):
        pages = -(-context // 16)
        keys, values = rand(pages + 1, kv_heads, 16, 128), rand(pages + 1, kv_heads, 128, 16)
        q = rand(q_tokens, q_heads * 128)
        out = torch.empty(q_tokens, q_heads * 128, dtype=torch.bfloat16, device=device)
        cu = torch.tensor([0, q_tokens], dtype=torch.int32, device=device)
        ctx = torch.tensor([context], dtype=torch.int32, device=device)
        table = torch.arange(pages, dtype=torch.int32, device=device).view(1, pages)
        return lambda: ops.paged_attention(q, keys, values, out, cu, ctx, table, num_seqs=1, max_q_len=q_tokens,
                                           q_heads=q_heads, kv_heads=kv_heads, head_dim=128, scale=128 ** -0.5,
                                           num_decode=1 if q_tokens == 1 else 0, max_ctx=context)

    # causal attention of a 128-token prompt, 8 heads of 128 (the reference's [1, 8, 128, 128]), over the paged cache
    record["causal_prefill_1x8x128x128"] = dict(measure(paged(128, 128, 8, 8)), reference_l4_ms=0.0891)
    # one decoded token over 127 cached keys and its own, 32 query heads, 8 kv heads of 128, pages of 16
    record["paged_gqa_decode_past127_q32_kv8"] = dict(measure(paged(128, 1, 32, 8)), reference_l4_ms=0.1004)

    # beside the reference's three: a sampling call for 8 and 64 rows of a 151,936-token vocabulary with
    # temperature, top-k, top-p and min-p (parameters packed and sent, the kernel's launches, tokens read back)
    from forge_engine_amd.sampling import SamplingParams
    from forge_engine_amd.sampling.sampler import Sampler

    sampler = Sampler(device)
    for rows in (8, 64):
        logits = rand(rows, 151936, dtype=torch.float32) * 3
        params = [SamplingParams(temperature=0.8, top_k=50, top_p=0.9, min_p=0.05, seed=1)] * rows
        seeds, draws = list(range(rows)), [3] * rows
        record[f"sample_top_k_top_p_min_p_{rows}x151936"] = measure(lambda: sampler.sample(logits, params, seeds, draws))
    print(json.dumps(record))
    return 0


def cross_check(args) -> int:
    """The model at the benchmark's sizes in bfloat16 against the same weights in 32-bit: a
    prompt whole (logits at a place in its middle and at its end), then eight single tokens.
    Rounding grows slowly with the number of layers; a kernel that is wrong at these sizes
    only (a width, a head count, a cache of this length) shows as a jump."""
    import torch

    from forge_engine_amd.config import load_model_config
    from forge_engine_amd.engine import ModelRunner, StepEntry, random_model

    chosen = MODELS[args.model]
    raw = dict(chosen["config"])
    full_layers = raw["num_hidden_layers"]
    if args.layers is not None:
        raw["num_hidden_layers"] = args.layers
    config = load_model_config(raw)
    prompt = args.prefill_tokens
    generator = torch.Generator().manual_seed(args.seed)
    tokens = torch.randint(0, config.vocab_size, (prompt + 8,), generator=generator).tolist()
    rows = {}
    for dtype in ("bfloat16", "float32"):
        model = random_model(config, args.seed, dtype=dtype, device=torch.device("cuda:0"))
        runner = ModelRunner(model, block_size=args.block_size,
                             block_capacity=-(-(prompt + 8) // args.block_size) + 1, num_state_slots=2)
        runner.begin("a")
        got = [runner.step([StepEntry("a", tokens[:prompt], [prompt // 2, prompt - 1])]).float().cpu()]
        for token in tokens[prompt:]:
            got.append(runner.step([StepEntry("a", [token], [0])]).float().cpu())
        rows[dtype] = torch.cat(got)
        del runner, model
        torch.cuda.empty_cache()
    want, got = rows["float32"], rows["bfloat16"]
    scale = float(want.abs().max())
    apart = (got - want).abs().max(dim=1).values
    print(json.dumps({
        "check": "bfloat16 against float32", "model": chosen["label"], "layers_run": config.num_hidden_layers,
        "layers_model": full_layers, "prompt_tokens": prompt, "rows": len(apart), "largest_logit": round(scale, 3),
        "largest_difference": round(float(apart.max()), 4), "fraction": round(float(apart.max()) / scale, 4),
        "argmax_agree": int((got.argmax(1) == want.argmax(1)).sum()),
    }))
    return 0


def design_configs(width: int, layers: int) -> dict:
    """Mazanex and Qwen3 at one width with layers of equal size: heads of 128, a group of four, a
    feed-forward three times the width, the same vocabulary and layer count.  Mazanex cycles through
    its three mixers (parallel attention + RWKV, gated linear attention, mLSTM)."""
    heads = max(4, width // 128)
    attention = {"heads": heads, "kv_heads": heads // 4, "dim": 128, "vdim": 128, "conv": 4, "mask": {"size": 2048},
                 "rot": {"dims": 64, "base": 10000.0}, "scale": 128 ** -0.5}
    mixers = [("parallel", {"left": attention, "right": {"heads": width // 64, "dim": 64, "rank": 64}}),
              ("gla", {"heads": heads, "dim": 64, "vdim": 128, "tau": 16.0, "rank": 16}),
              ("mlstm", {"heads": max(2, heads // 2), "dim": 128, "vdim": 256, "gate_cap": 15.0})]
    mazanex = {"architecture": "Mazanex", "vocab": 32000, "width": width, "norm": {"eps": 1e-6},
               "layers": [{"type": mixers[i % 3][0], "mixer": mixers[i % 3][1], "mlp": {"kind": "dense", "ff": 3 * width}}
                          for i in range(layers)]}
    qwen3 = _qwen3(vocab_size=32000, hidden_size=width, intermediate_size=3 * width, num_hidden_layers=layers,
                   num_attention_heads=heads, num_key_value_heads=heads // 4, rope_theta=1000000.0,
                   tie_word_embeddings=False, eos_token_id=None)
    return {"Mazanex": mazanex, "Qwen3": qwen3}


def rekezen_configs(width: int, layers: int) -> dict:
    """Rekezen and Qwen3 at one width: heads of 128 in groups of four, the same vocabulary and layer
    count.  Rekezen's feed-forward is a mixture of eight experts as wide as the model, of which a token
    takes two, beside a shared one of the same size: three widths of active feed-forward a token, as
    many as Qwen3's dense one.  Every second layer reads the keys and values of the layer before it;
    four residual streams; a table of token pairs beside the embedding."""
    heads = max(4, width // 128)

    def mixer(index):
        sizes = {"heads": heads, "kv_heads": heads // 4, "dim": 128, "vdim": 128, "scale": 128 ** -0.5, "softcap": 30.0,
                 "rot": {"dims": 64, "base": 100000.0, "scaling": {"factor": 8.0, "original": 4096, "fast": 32.0, "slow": 1.0}}}
        if index % 2:
            sizes["kv_from"] = index - 1
        return sizes

    mlp = {"kind": "moe", "router": {"experts": 8, "top": 2}, "expert": {"ff": width, "limit": 7.0},
           "shared": {"ff": width, "limit": 7.0}}
    rekezen = {"architecture": "Rekezen", "vocab": 32000, "width": width, "norm": {"eps": 1e-6}, "streams": 4,
               "embedding": {"bigram": {"buckets": 65521, "mul_prev": 36313, "mul_cur": 27191}}, "logit_scale": 1.0,
               "layers": [{"type": "attention", "mixer": mixer(i), "mlp": mlp} for i in range(layers)]}
    return {"Rekezen": rekezen, "Qwen3": design_configs(width, layers)["Qwen3"]}


def malusun_configs(width: int, layers: int) -> dict:
    """Malusun beside Rekezen (the closest existing model: attention over the general path and a mixture of experts
    beside a shared one) and Qwen3, at one width: heads of 128 in groups of four, the same vocabulary and layer
    count.  Malusun cycles through its three mixers: the selective scan (twice the width inside, 16 states a
    channel, a step size of rank width / 16, four taps) with the dense feed-forward of three widths, then rotary
    and penalised attention over windows of 1,024 with eight experts as wide as the model of which a token takes
    two, beside a shared one of the same size; values lean on the first attention layer's."""
    heads = max(4, width // 128)
    attention = {"heads": heads, "kv_heads": heads // 4, "dim": 128, "vdim": 128, "scale": 128 ** -0.5, "mask": {"size": 1024},
                 "v_mix": True}
    moe = {"kind": "moe", "router": {"experts": 8, "top": 2}, "expert": {"ff": width}, "shared": {"ff": width}}
    kinds = [("mamba1", {"inner": 2 * width, "state": 16, "dt_rank": max(8, width // 16), "conv": 4}, {"kind": "dense", "ff": 3 * width}),
             ("attention", dict(attention, rot={"dims": 64, "base": 500000.0}), moe),
             ("attention_2", attention, moe)]
    malusun = {"architecture": "Malusun", "vocab": 32000, "width": width, "norm": {"eps": 1e-6}, "embedding": {"scale": 0.5},
               "layers": [{"type": kinds[i % 3][0], "mixer": kinds[i % 3][1], "mlp": kinds[i % 3][2]} for i in range(layers)]}
    others = rekezen_configs(width, layers)
    return {"Malusun": malusun, "Rekezen": others["Rekezen"], "Qwen3": others["Qwen3"]}


def dubizen_configs(width: int, layers: int) -> dict:
    """Dubizen beside Rekezen (the closest existing model: attention over the general path, layers that read an
    earlier layer's cache, layer norms, a mixture of experts beside a shared one) and Qwen3, at one width: heads of
    128, the same vocabulary and layer count.  Dubizen cycles through attention over a latent (a cached row of 512
    + 64 numbers a token, queries through a bottleneck of 3/8 of the width, 64 rotated dims a head) with the dense
    feed-forward of three widths, attention over a window of 1,024 in groups of four with biases by distance and
    eight experts as wide as the model of which a token takes two out of the two best of four groups, beside a
    gated shared one, and a layer that reads the first one's cache with the same experts."""
    heads = max(4, width // 128)
    latent = {"heads": heads, "dim": 128, "rot_dim": 64, "vdim": 128, "q_rank": max(128, 3 * width // 8), "kv_rank": 512,
              "scale": 192 ** -0.5, "rot": {"dims": 64, "base": 10000.0}}
    windowed = {"heads": heads, "kv_heads": heads // 4, "dim": 128, "vdim": 128, "scale": 128 ** -0.5, "mask": {"size": 1024},
                "bias_max": 512.0, "bias_rows": 32}
    moe = {"kind": "moe", "router": {"experts": 8, "top": 2, "scale": 2.0, "groups": {"count": 4, "keep": 2}}, "expert": {"ff": width},
           "shared": {"ff": width}}

    def entry(index):
        if index % 3 == 0:
            return {"type": "latent_attention", "mixer": latent, "mlp": {"kind": "dense", "ff": 3 * width}}
        if index % 3 == 1:
            return {"type": "attention", "mixer": windowed, "mlp": moe}
        return {"type": "latent_attention", "mixer": dict(latent, kv_from=index - 2), "mlp": moe}

    dubizen = {"architecture": "Dubizen", "vocab": 32000, "width": width, "norm": {"eps": 1e-6}, "residual_mult": 0.5,
               "layers": [entry(i) for i in range(layers)]}
    others = rekezen_configs(width, layers)
    return {"Dubizen": dubizen, "Rekezen": others["Rekezen"], "Qwen3": others["Qwen3"]}


def talapel_configs(width: int, layers: int) -> dict:
    """Talapel beside Mazanex (mixers side by side, recurrences over a matrix state), Malusun (a state-space scan, a
    mixture of experts) and Qwen3, at one width: heads of 128 in groups of four, the same vocabulary, as many layer
    runs as the others have layers.  Talapel passes twice through half as many layers: capped attention beside a
    state-space recurrence (twice the width inside, heads of 64, 128 states, eight groups) with the dense feed-forward
    of three widths, retention (keys of 128, values of 256), attention beside the recurrence again, both with eight
    experts as wide as the model of which a token's id names two."""
    heads = max(4, width // 128)
    side = {"left": {"heads": heads, "kv_heads": heads // 4, "dim": 128, "vdim": 128, "scale": 128 ** -0.5, "softcap": 30.0,
                     "q_temp": {"coef": 0.5, "every": 512}},
            "right": {"heads": width // 32, "vdim": 64, "state": 128, "groups": 8, "conv": 4, "norm_groups": 8},
            "left_scale": 1.2, "right_scale": 0.8}
    keep = {"heads": heads, "dim": 128, "vdim": 256, "decay": [1.0 - 2.0 ** -(5 + h % 6) for h in range(heads)],
            "rot": {"dims": 128, "base": 10000.0}}
    moe = {"kind": "moe", "router": {"experts": 8, "top": 2}, "expert": {"ff": width}}
    kinds = [("parallel", side, {"kind": "dense", "ff": 3 * width}), ("retention", keep, moe), ("parallel", side, moe)]
    own = max(1, layers // 2)
    talapel = {"architecture": "Talapel", "vocab": 32000, "width": width, "norm": {"eps": 1e-6}, "embedding": {"scale": width ** 0.5},
               "loop": {"start": 0, "stop": own, "times": 2},
               "layers": [{"type": kinds[i % 3][0], "mixer": kinds[i % 3][1], "mlp": kinds[i % 3][2]} for i in range(own)]}
    others = dict(design_configs(width, layers), Malusun=malusun_configs(width, layers)["Malusun"])
    return {"Talapel": talapel, "Mazanex": others["Mazanex"], "Malusun": others["Malusun"], "Qwen3": others["Qwen3"]}


def budanex_configs(width: int, layers: int) -> dict:
    """Budanex beside Dubizen (attention through a latent), Talapel (passes, the state-space recurrence, capped attention),
    Rekezen (norms over whole projections) and Qwen3, at one width: heads of 128, the same vocabulary, as many layer runs
    as the others have layers.  Budanex passes twice through half as many layers: softcapped attention in groups of four
    with half of every head turned, a state-space recurrence (twice the width inside, heads of 64, 128 states, eight
    groups), attention through a latent (a cached row of 512 + 64 numbers a token) over a window of 1,024; every layer
    with the gated feed-forward of three widths."""
    heads = max(4, width // 128)
    attention = {"heads": heads, "kv_heads": heads // 4, "dim": 128, "vdim": 128, "scale": 128 ** -0.5, "softcap": 30.0,
                 "rot": {"dims": 64, "base": 10000.0}}
    recurrence = {"heads": width // 32, "vdim": 64, "state": 128, "groups": 8, "conv": 4, "norm_groups": 8}
    latent = {"heads": heads, "dim": 128, "rot_dim": 64, "vdim": 128, "kv_rank": 512, "scale": 192 ** -0.5, "mask": {"size": 1024},
              "rot": {"dims": 64, "base": 100000.0, "scaling": {"factor": 8.0, "original": 4096, "fast": 32.0, "slow": 1.0}}}
    kinds = [("attention", attention), ("mamba2", recurrence), ("latent_attention", latent)]
    own = max(1, layers // 2)
    budanex = {"architecture": "Budanex", "vocab": 32000, "width": width, "norm": {"eps": 1e-6}, "logit_softcap": 30.0,
               "loop": {"start": 0, "stop": own, "times": 2},
               "layers": [{"type": kinds[i % 3][0], "mixer": kinds[i % 3][1], "mlp": {"kind": "dense", "ff": 3 * width}} for i in range(own)]}
    others = dubizen_configs(width, layers)
    return {"Budanex": budanex, "Dubizen": others["Dubizen"], "Talapel": talapel_configs(width, layers)["Talapel"],
            "Rekezen": others["Rekezen"], "Qwen3": others["Qwen3"]}


DESIGN_CONFIGS = {"mazanex": design_configs, "rekezen": rekezen_configs, "malusun": malusun_configs, "dubizen": dubizen_configs,
                  "talapel": talapel_configs, "budanex": budanex_configs}


def design_comparison(args) -> int:
    """Prefill and decode throughput of Mazanex (or, with ``--design``, Rekezen, Malusun, Dubizen, Talapel or Budanex) beside the closest existing models at equal
    width, layer count, feed-forward size and vocabulary; random weights, one JSON line a model and width."""
    import torch

    from forge_engine_amd.config import load_model_config
    from forge_engine_amd.engine import ModelRunner, StepEntry, random_model

    device = torch.device("cuda:0")
    dtype = {"bf16": "bfloat16", "fp32": "float32"}[args.dtype]
    layers = args.layers or 6
    batch = args.batch or 8
    prompt_len = args.prompt_len or 1024
    generator = torch.Generator().manual_seed(args.seed)
    for width in (int(w) for w in args.widths.split(",")):
        for label, raw in DESIGN_CONFIGS[args.design](width, layers).items():
            if args.only and label.lower() != args.only.lower():
                continue
            config = load_model_config(raw)
            model = random_model(config, args.seed, dtype=dtype, device=device)
            pages = -(-(max(args.prefill_tokens, prompt_len) + args.steps + args.warmup + 16) // args.block_size)
            runner = ModelRunner(model, block_size=args.block_size, block_capacity=(batch + 1) * pages,
                                 num_state_slots=batch + 1, eager_sightings=1)
            vocab = raw.get("vocab", raw.get("vocab_size"))

            def tokens(n):
                return torch.randint(0, vocab, (n,), generator=generator).tolist()

            def time_ms(fn, warmup, steps):
                for _ in range(warmup):
                    fn()
                torch.cuda.synchronize()
                events = [(torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)) for _ in range(steps)]
                for begin, end in events:
                    begin.record()
                    fn()
                    end.record()
                torch.cuda.synchronize()
                return spread([begin.elapsed_time(end) for begin, end in events])["median"]

            prompt = tokens(args.prefill_tokens)

            def prefill_once():
                runner.begin("p")
                runner.step([StepEntry("p", prompt, [len(prompt) - 1])])
                runner.end("p")

            prefill_ms = time_ms(prefill_once, 2, max(3, min(10, args.steps)))
            names = [f"d{i}" for i in range(batch)]
            for name in names:
                runner.begin(name)
                runner.step([StepEntry(name, tokens(prompt_len), [])])
            # different tokens: a design may choose experts by the token's id
            entries = [StepEntry(name, [token], [0]) for name, token in zip(names, tokens(batch))]
            decode_ms = time_ms(lambda: runner.step(entries), args.warmup, args.steps)
            print(json.dumps({
                "phase": "design", "model": label, "width": width, "layers": layers, "dtype": args.dtype,
                "weight_gb": round(weight_bytes(model) / 1e9, 3),
                "prefill_tokens": args.prefill_tokens, "prefill_ms": prefill_ms,
                "prefill_tokens_per_s": round(args.prefill_tokens / prefill_ms * 1e3, 1),
                "decode_batch": batch, "decode_context": prompt_len, "decode_ms": decode_ms,
                "decode_tokens_per_s": round(batch / decode_ms * 1e3, 1),
                "graph_replays": runner.graph_replays,
            }), flush=True)
            del runner, model
            torch.cuda.empty_cache()
    return 0


def main() -> int:
    args = parse_args()
    if args.gpus != 1:
        print(f"bench.py measures one GPU; --gpus {args.gpus} is not supported by this engine")
        return 2
    if args.phase == "micro":
        return micro_benchmarks()
    if args.phase == "check":
        return cross_check(args)
    if args.phase == "design":
        return design_comparison(args)
    import torch

    from forge_engine_amd.config import SchedulerConfig, load_model_config
    from forge_engine_amd.engine import ModelRunner, StepEntry, random_model
    from forge_engine_amd.engine.scheduler import ConcurrentGenerationEngine
    from forge_engine_amd.sampling import SamplingParams
    from forge_engine_amd.sampling.sampler import Sampler

    chosen = MODELS[args.model]
    raw = dict(chosen["config"])
    full_layers = raw["num_hidden_layers"]
    if args.layers is not None:
        raw["num_hidden_layers"] = args.layers
    config = load_model_config(raw)
    device = torch.device("cuda:0")
    dtype = {"bf16": "bfloat16", "fp32": "float32"}[args.dtype]

    def timed(fn, warmup, steps):
        """Per-step device times (ms) of ``steps`` calls after ``warmup`` untimed ones, and the
        host's mean over the same calls."""
        for _ in range(warmup):
            fn()
        torch.cuda.synchronize()
        events = [(torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)) for _ in range(steps)]
        start = time.perf_counter()
        for begin, end in events:
            begin.record()
            fn()
            end.record()
        torch.cuda.synchronize()
        wall = (time.perf_counter() - start) / steps
        return [begin.elapsed_time(end) for begin, end in events], wall * 1e3

    def measured_read_bandwidth() -> float:
        """Bytes a second of a plain streaming read: a kernel that only reads, over four 400 MB
        buffers in turn so that no cache holds what it reads, twenty times between one pair of
        device events."""
        from forge_engine_amd.kernels import ops

        buffers = [torch.zeros(100_000_000, dtype=torch.float32, device=device) for _ in range(4)]
        sink = torch.zeros(1, dtype=torch.float32, device=device)
        for data in buffers:
            ops.stream_read(data, sink)
        begin, end = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
        begin.record()
        for index in range(20):
            ops.stream_read(buffers[index % 4], sink)
        end.record()
        torch.cuda.synchronize()
        seconds = begin.elapsed_time(end) * 1e-3 / 20
        return 400_000_000 / seconds

    read_peak = measured_read_bandwidth()
    model = random_model(config, args.seed, dtype=dtype, device=device)
    sampler = Sampler(device)
    greedy = SamplingParams()
    generator = torch.Generator().manual_seed(args.seed)

    def random_tokens(n):
        return torch.randint(0, config.vocab_size, (n,), generator=generator).tolist()

    element = 2 if args.dtype == "bf16" else 4
    layers = config.num_hidden_layers
    kv_bytes_per_token = 2 * layers * config.kv_size * element

    if args.workload == "mixed":
        low, high = (int(v) for v in args.prompt_range.split(","))
        lengths = torch.randint(low, high + 1, (args.requests,), generator=generator).tolist()
        pages = sum(-(-(n + args.new_tokens) // args.block_size) for n in lengths)
        runner = ModelRunner(model, block_size=args.block_size, block_capacity=pages, num_state_slots=args.requests)
        scheduler = SchedulerConfig(max_requests=args.requests, max_batch_size=min(64, args.requests),
                                    token_budget=args.token_budget, block_size=args.block_size, block_capacity=pages,
                                    max_context=args.context)
        engine = ConcurrentGenerationEngine(runner, sampler, greedy, scheduler, eos_token_ids=())
        for round_index in range(2):        # the first round warms up (graphs are captured), the second is timed
            ids = [engine.submit(random_tokens(n), sampling_params=SamplingParams(max_new_tokens=args.new_tokens))
                   for n in lengths]
            torch.cuda.synchronize()
            start = time.perf_counter()
            steps = 0
            while not engine.idle:
                engine.step()
                steps += 1
            torch.cuda.synchronize()
            seconds = time.perf_counter() - start
            for request_id in ids:
                engine.forget(request_id)
        generated = args.requests * args.new_tokens
        print(json.dumps({
            "workload": "mixed", "through": "scheduler", "model": chosen["label"], "dtype": args.dtype,
            "requests": args.requests, "prompt_tokens": sum(lengths), "generated_tokens": generated,
            "token_budget": args.token_budget, "steps": steps, "seconds": round(seconds, 3),
            "generated_tokens_per_s": round(generated / seconds, 1),
            "all_tokens_per_s": round((generated + sum(lengths)) / seconds, 1),
            "layers_run": layers, "layers_model": full_layers,
        }))
        return 0

    batches = sorted({args.batch, *[int(b) for b in args.points.split(",") if b]})
    if args.phase == "decode" or args.through == "scheduler":
        batches = [args.batch]
    spare = args.steps + args.warmup + 8
    # through the scheduler the first requests already decode while the last prompts are still fed
    joining = max(batches) * args.prompt_len // max(args.token_budget, 1) + 2 if args.through == "scheduler" else 0
    spare += joining
    per_request = -(-(args.prompt_len + spare) // args.block_size)
    capacity = max(args.batch * -(-args.context // args.block_size), max(batches) * per_request,
                   -(-(args.prefill_tokens + 1) // args.block_size))
    runner = ModelRunner(model, block_size=args.block_size, block_capacity=capacity,
                         num_state_slots=max(batches) + 1, eager_sightings=1)   # the timed loops repeat one shape

    def decode_run(batch):
        names = [f"d{batch}_{i}" for i in range(batch)]
        state = {}
        for name in names:
            runner.begin(name)
            prompt = random_tokens(args.prompt_len)
            for at in range(0, len(prompt), 2048):      # untimed: fill the cache
                portion = prompt[at:at + 2048]
                last = at + 2048 >= len(prompt)
                logits = runner.step([StepEntry(name, portion, [len(portion) - 1] if last else [])])
            state[name] = sampler.sample(logits, [greedy], [0], [0])[0]

        def one_step():
            logits = runner.step([StepEntry(n, [state[n]], [0]) for n in names])
            tokens = sampler.sample(logits, [greedy] * batch, [0] * batch, [0] * batch)
            for n, t in zip(names, tokens):
                state[n] = t

        # The sampled tokens go into the next step on the device, and the host reads them while
        # that step runs (a step late): the GPU does not wait for the host between two steps.
        placeholders = [StepEntry(n, [0], [0]) for n in names]
        flight = {"feed": torch.tensor([state[n] for n in names], dtype=torch.int32, device=device), "unread": None}

        def one_overlapped_step():
            logits = runner.step(placeholders, device_tokens=flight["feed"])
            both = sampler.sample_greedy_on_device(logits)
            if flight["unread"] is not None:
                sampler.read(flight["unread"])
            flight["unread"], flight["feed"] = both, both[0]

        overlapped = args.overlap and runner.feeds_from_device(placeholders)
        times, wall = timed(one_overlapped_step if overlapped else one_step, args.warmup, args.steps)
        contexts = [runner.length(n) for n in names]
        for name in names:
            runner.end(name)
        return times, wall, sum(contexts) / batch - args.steps / 2.0

    def scheduler_run(batch):
        """The same decode steps through the scheduler: requests are admitted with their prompts,
        stepped until every one decodes, then K calls of step() are timed."""
        scheduler = SchedulerConfig(max_requests=batch, max_batch_size=batch, token_budget=max(args.token_budget, batch),
                                    block_size=args.block_size, block_capacity=capacity, overlap_decode=args.overlap)
        engine = ConcurrentGenerationEngine(runner, sampler, greedy, scheduler, eos_token_ids=())
        limit = args.steps + args.warmup + 4 + joining
        drawn = dict(temperature=0.8, top_k=50, top_p=0.9) if args.sampled else {}
        ids = [engine.submit(random_tokens(args.prompt_len), sampling_params=SamplingParams(max_new_tokens=limit, seed=i, **drawn))
               for i in range(batch)]
        while any(n != 1 for n in engine.snapshot().last_batch_tokens) or len(engine.snapshot().last_batch) != batch:
            engine.step()
        times, wall = timed(engine.step, args.warmup, args.steps)
        mean_ctx = sum(runner.length(request_id) for request_id in ids) / batch - args.steps / 2.0
        for request_id in ids:
            engine.cancel(request_id)
        return times, wall, mean_ctx

    run = scheduler_run if args.through == "scheduler" else decode_run
    results = {} if args.phase == "prefill" else {b: run(b) for b in batches}

    # prefill: one whole prompt in one step, logits at its last token
    prompt = random_tokens(args.prefill_tokens)
    counter = [0]

    def prefill_once():
        name = f"p{counter[0]}"
        counter[0] += 1
        runner.begin(name)
        logits = runner.step([StepEntry(name, prompt, [len(prompt) - 1])])
        sampler.sample(logits, [greedy], [0], [0])
        runner.end(name)

    def roofline(batch, times, mean_ctx):
        seconds = spread(times)["median"] * 1e-3
        step_bytes = weight_bytes(model) + batch * mean_ctx * kv_bytes_per_token
        achieved = step_bytes / seconds
        return {"bound": "hbm", "achieved": round(achieved / 1e9, 1), "peak": HBM_BYTES_PER_S / 1e9, "unit": "GB/s",
                "frac": round(achieved / HBM_BYTES_PER_S, 4), "measured_peak": round(read_peak / 1e9, 1),
                "frac_measured": round(achieved / read_peak, 4)}

    if args.phase == "decode" or args.through == "scheduler":
        times, wall, mean_ctx = results[args.batch]
        median = spread(times)["median"]
        print(json.dumps({"phase": "decode", "through": args.through, "model": chosen["label"], "batch": args.batch,
                          "ms_per_step": median, "ms_per_step_wall": round(wall, 4), "step_ms": spread(times),
                          "value": round(args.batch / median * 1e3, 2), "unit": "tokens/s",
                          "roofline": roofline(args.batch, times, mean_ctx),
                          "layers_run": layers, "layers_model": full_layers}))
        return 0
    prefill_times, _ = timed(prefill_once, 2, max(3, min(10, args.steps)))
    prefill_ms = spread(prefill_times)["median"]
    matrix_params = layers * (config.hidden_size * (config.q_size + 2 * config.kv_size)
                              + config.q_size * config.hidden_size
                              + 3 * config.hidden_size * config.intermediate_size)
    t = args.prefill_tokens
    prefill_flops = 2.0 * t * matrix_params + 2.0 * t * t * config.q_size * layers \
        + 2.0 * config.vocab_size * config.hidden_size
    if args.phase == "prefill":
        print(json.dumps({"phase": "prefill", "model": chosen["label"], "dtype": args.dtype, "tokens": t, "ms": prefill_ms,
                          "step_ms": spread(prefill_times),
                          "value": round(t / prefill_ms * 1e3, 1), "unit": "tokens/s",
                          "frac": round(prefill_flops / (prefill_ms * 1e-3) / PEAK_FLOPS[args.dtype], 4),
                          "peak_tflops": PEAK_FLOPS[args.dtype] / 1e12,
                          "layers_run": layers, "layers_model": full_layers}))
        return 0

    times, wall, mean_ctx = results[args.batch]
    median = spread(times)["median"]
    record = {
        "metric": f"decode tok/s at batch {args.batch} ({chosen['label']} sizes, {args.prompt_len}-token prompts)",
        "value": round(args.batch / median * 1e3, 2),
        "unit": "tokens/s",
        "n_gpus": 1,
        "steps": args.steps,
        "warmup": args.warmup,
        "ms_per_step": median,
        "ms_per_step_wall": round(wall, 4),
        "step_ms": spread(times),
        "higher_is_better": True,
        "scaling": "weak",
        "vs_baseline": None,
        "dtype": args.dtype,
        "data": "synthetic: random weights drawn on the device, uniform-random token ids",
        "config": {
            "model": f"{chosen['label']} sizes (Qwen3ForCausalLM)", "global_batch": args.batch,
            "seq_len": args.prompt_len, "parallelism": "single GPU", "context": args.context,
            "block_size": args.block_size, "layers_run": layers, "layers_model": full_layers,
            "hidden_size": config.hidden_size, "intermediate_size": config.intermediate_size,
            "q_heads": config.num_attention_heads, "kv_heads": config.num_key_value_heads,
            "head_dim": config.head_dim, "vocab_size": config.vocab_size,
            "tied_embeddings": config.tie_word_embeddings, "rope_theta": config.rope_theta,
            "prefill_tokens": args.prefill_tokens, "sampling": "greedy",
        },
        "prefill": {
            "value": round(t / prefill_ms * 1e3, 1), "tokens": t, "ms": prefill_ms,
            "frac": round(prefill_flops / (prefill_ms * 1e-3) / PEAK_FLOPS[args.dtype], 4),
        },
        "roofline": roofline(args.batch, times, mean_ctx),
        "points": {f"decode_b{b}": round(b / spread(results[b][0])["median"] * 1e3, 2) for b in batches if b != args.batch},
    }
    print(json.dumps(record))
    return 0


if __name__ == "__main__":
    raise SystemExit(main())
