"""`bench.py --ritevik`: prefill and decode throughput of Ritevik at two sizes of a real model's layers (random weights),
beside the framework's closest existing model, the int4 GPT-2, at the same width, heads, feed-forward and layer runs.

Both models run the same steps through the same calls: prefill of prompts from an empty cache (generate_cached with one new
token, the runtime's own events around the prompt's forward), decode steps as the runtime replays them (decode_steps).
Every figure is the best of a few repetitions; the two models take turns.  `weight_bytes` are the bytes of weights a decode step
reads (embedding tables left out); `hbm_frac` is weight_bytes plus the cache's bytes over the step's time and 8 TB/s."""
import json

import numpy as np

HBM_BYTES_PER_S = 8.0e12
SIZES = {"small": dict(gpt2=dict(n_layer=12, n_embd=768, n_head=12, vocab=50257), prompts=(128, 1024, 2048), positions=2304),
         "large": dict(gpt2=dict(n_layer=24, n_embd=2048, n_head=32, vocab=50257), prompts=(128, 1024, 4096), positions=4608)}
DECODE = ((1, 1024), (4, 1024), (16, 1024))  # batch, context


def gpt2_random_int4(cfg, n_positions, group, seed):
    """The dict of workloads.quantize_gpt2 with nibbles drawn directly (cut from one pool), scales and LayerNorms constant."""
    rng = np.random.default_rng(seed)
    pool = rng.integers(0, 1 << 32, 1 << 22, dtype=np.uint32)
    d, V = cfg["n_embd"], cfg["vocab"]

    def lin(K, N, bias=True):
        packed = np.resize(np.roll(pool, -int(rng.integers(0, pool.size)))[: min(pool.size, K // 8 * N)], (K // 8, N))
        return packed, np.full(((K + group - 1) // group, N), 0.2 / np.sqrt(K), np.float32), np.zeros(N, np.float32) if bias else None

    one, zero = np.ones(d, np.float32), np.zeros(d, np.float32)
    layers = [dict(ln1_g=one, ln1_b=zero, ln2_g=one, ln2_b=zero, qkv=lin(d, 3 * d), proj=lin(d, d), fc=lin(d, 4 * d), fc_proj=lin(4 * d, d))
              for _ in range(cfg["n_layer"])]
    head = lin(d, V, False)
    wte = np.resize(rng.standard_normal(1 << 20, dtype=np.float32) * np.float32(0.02), (V, d))
    return dict(group=group, wte=wte, wpe=np.resize(wte, (n_positions, d)), lnf_g=one, lnf_b=zero, layers=layers, lm_head=(head[0], head[1]))


def step_weight_bytes_ritevik(model, spec):
    """Weight bytes of one step's layer runs and head (looped layers count once per pass), embedding tables left out."""
    per = {}
    for name, rows, cols, _ in model.tensor_list():
        key = name.split(".")[0]
        per[key] = per.get(key, 0) + 2 * rows * cols
    loop = spec.get("loop")
    total = per["head"]
    for i in range(len(spec["layers"])):
        total += per[f"l{i}"] * (loop["times"] if loop and loop["start"] <= i < loop["stop"] else 1)
    return total + (2 * 2 * spec["width"] ** 2 * loop["times"] if loop else 0)


def cache_bytes_ritevik(spec, context):
    """Bytes a step of one sequence reads and writes in caches and states."""
    loop, total = spec.get("loop"), 0
    for i, e in enumerate(spec["layers"]):
        m, n = e["mixer"], loop["times"] if loop and loop["start"] <= i < loop["stop"] else 1
        if e["type"] == "latent_attention":
            total += n * 2 * context * (m["kv_rank"] + m["rot_dim"])
        else:
            total += n * 2 * 4 * m["heads"] * m["dim"] * m["vdim"]
    return total


def measure(model, vocab, prompts, seed=0):
    rng = np.random.default_rng(seed)
    out = {"prefill_ms": {}, "decode_ms": {}}
    for n in prompts:
        p = rng.integers(0, vocab, (1, n)).astype(np.uint32)
        out["prefill_ms"][n] = min(model.generate_cached(p, 1, eos=-1)[1][0] for _ in range(4))
    for B, context in DECODE:
        p = rng.integers(0, vocab, (B, context)).astype(np.uint32)
        model.reset_cache()
        model.forward_cached(p, all_rows=False)
        model.decode_steps(B, 8)
        out["decode_ms"][B] = min(model.decode_steps(B, 24) / 24 for _ in range(3))
    return out


def trace(model, vocab, context=1024, batch=16):
    """A short run for kernel traces: three prefills, then decode steps launched one by one, of one sequence and of a batch."""
    rng = np.random.default_rng(0)
    model.set_decode_mode(model.DECODE_EAGER)
    for _ in range(3):
        model.reset_cache()
        model.forward_cached(rng.integers(0, vocab, (1, context)), all_rows=False)
    model.decode_steps(1, 32)
    model.reset_cache()
    model.forward_cached(rng.integers(0, vocab, (batch, context)), all_rows=False)
    model.decode_steps(batch, 16)


def run(sizes, trace_model=None, context=1024, emit=lambda d: print(json.dumps(d), flush=True)):
    from async_gpu_amd import gpt2, ritevik, workloads
    rows = []
    for size in sizes:
        c = SIZES[size]
        spec = workloads.RITEVIK_SMALL if size == "small" else workloads.RITEVIK_LARGE
        g = c["gpt2"]
        if trace_model == "gpt2":
            gm = gpt2.Int4Gpt2Model.from_quantized(gpt2.Gpt2Config(g["n_layer"], g["n_embd"], g["n_head"], vocab_size=g["vocab"], n_positions=c["positions"],
                                                                   group_size=32, max_batch=16), gpt2_random_int4(g, c["positions"], 32, 1))
            trace(gm, g["vocab"], context)
            gm.close()
            continue
        rm = ritevik.RitevikModel.from_tensors(spec, workloads.ritevik_tensors(spec, 1), n_positions=c["positions"], max_batch=16)
        if trace_model == "ritevik":
            trace(rm, spec["vocab"], context)
            rm.close()
            continue
        gm = gpt2.Int4Gpt2Model.from_quantized(gpt2.Gpt2Config(g["n_layer"], g["n_embd"], g["n_head"], vocab_size=g["vocab"], n_positions=c["positions"],
                                                               group_size=32, max_batch=16), gpt2_random_int4(g, c["positions"], 32, 1))
        both = {"ritevik": measure(rm, spec["vocab"], c["prompts"]), "gpt2_int4": measure(gm, g["vocab"], c["prompts"])}
        d = g["n_embd"]
        wb = {"ritevik": step_weight_bytes_ritevik(rm, spec), "gpt2_int4": int((g["n_layer"] * 12 * d * d + d * g["vocab"]) * (0.5 + 4.0 / 32))}
        for name, m in both.items():
            for B, context in DECODE:
                cb = B * (cache_bytes_ritevik(spec, context) if name == "ritevik" else g["n_layer"] * 2 * d * 4 * context)
                ms = m["decode_ms"][B]
                rows.append(dict(size=size, model=name, what="decode", batch=B, context=context, ms_per_step=round(ms, 4), tok_s=round(B * 1e3 / ms, 1),
                                 weight_bytes=wb[name], cache_bytes=cb, hbm_frac=round((wb[name] + cb) / (ms * 1e-3) / HBM_BYTES_PER_S, 4)))
            for n, ms in m["prefill_ms"].items():
                rows.append(dict(size=size, model=name, what="prefill", batch=1, tokens=n, ms=round(ms, 3), tok_s=round(n * 1e3 / ms, 1)))
        rm.close()
        gm.close()
    if trace_model:
        return
    head = [r for r in rows if r["model"] == "ritevik" and r["what"] == "decode" and r["batch"] == 1][0]
    emit({"metric": f"Ritevik decode tok/s (B=1, {head['size']} layers, bf16 weights)", "value": head["tok_s"], "unit": "tok/s", "n_gpus": 1,
          "higher_is_better": True, "vs_baseline": None, "dtype": "bf16 weights, f32 residual, scores and state", "data": "synthetic", "rows": rows})
