"""`bench.py --piralix`: prefill and decode throughput of Piralix at two sizes of a real model's layers (random weights), beside
the framework's closest existing model, Ritevik, at the same width, feed-forward, vocabulary and layer runs.  Both have bf16
weights and run the same steps through the same calls, as in `bench.py --ritevik`; the figures are defined there."""
import json

from bench_ritevik import DECODE, HBM_BYTES_PER_S, cache_bytes_ritevik, measure, step_weight_bytes_ritevik, trace

SIZES = {"small": dict(prompts=(128, 1024, 2048), positions=2304), "large": dict(prompts=(128, 1024, 4096), positions=4608)}


def passes(spec, i):
    loop = spec.get("loop")
    return loop["times"] if loop and loop["start"] <= i < loop["stop"] else 1


def step_weight_bytes(model, spec):
    """Weight bytes of one step's layer runs and head (the embedding table, read as a matrix)."""
    per = {}
    for name, rows, cols, _ in model.tensor_list():
        key = name.split(".")[0]
        per[key] = per.get(key, 0) + 2 * rows * cols
    return per["embed"] + sum(per[f"l{i}"] * passes(spec, i) for i in range(len(spec["layers"])))


def cache_bytes(spec, context):
    """Bytes a step of one sequence reads and writes in caches and states."""
    total = 0
    for i, e in enumerate(spec["layers"]):
        m = e["mixer"]
        if e["type"] == "attention":
            n = 2 * context * m["kv_heads"] * (m["dim"] + m["vdim"])
        elif e["type"] == "mlstm":
            n = 2 * 4 * m["heads"] * m["dim"] * (m["vdim"] + 1)
        else:
            n = 4 * m["width"] * (2 + m["conv"])
        total += n * passes(spec, i)
    return total


def run(sizes, trace_model=None, context=1024, emit=lambda d: print(json.dumps(d), flush=True)):
    from async_gpu_amd import piralix, ritevik, workloads
    rows = []
    for size in sizes:
        c = SIZES[size]
        specs = {"piralix": workloads.PIRALIX_SMALL if size == "small" else workloads.PIRALIX_LARGE,
                 "ritevik": workloads.RITEVIK_SMALL if size == "small" else workloads.RITEVIK_LARGE}
        make = {"piralix": lambda s: piralix.PiralixModel.from_tensors(s, workloads.piralix_tensors(s, 1), n_positions=c["positions"], max_batch=16),
                "ritevik": lambda s: ritevik.RitevikModel.from_tensors(s, workloads.ritevik_tensors(s, 1), n_positions=c["positions"], max_batch=16)}
        weight = {"piralix": step_weight_bytes, "ritevik": step_weight_bytes_ritevik}
        caches = {"piralix": cache_bytes, "ritevik": cache_bytes_ritevik}
        if trace_model:
            m = make[trace_model](specs[trace_model])
            trace(m, specs[trace_model]["vocab"], context)
            m.close()
            continue
        models = {name: make[name](specs[name]) for name in make}
        for name, m in models.items():
            got, wb = measure(m, specs[name]["vocab"], c["prompts"]), weight[name](m, specs[name])
            for B, n in DECODE:
                cb, ms = B * caches[name](specs[name], n), got["decode_ms"][B]
                rows.append(dict(size=size, model=name, what="decode", batch=B, context=n, ms_per_step=round(ms, 4), tok_s=round(B * 1e3 / ms, 1),
                                 weight_bytes=wb, cache_bytes=cb, hbm_frac=round((wb + cb) / (ms * 1e-3) / HBM_BYTES_PER_S, 4)))
            for n, ms in got["prefill_ms"].items():
                rows.append(dict(size=size, model=name, what="prefill", batch=1, tokens=n, ms=round(ms, 3), tok_s=round(n * 1e3 / ms, 1)))
        for m in models.values():
            m.close()
    if trace_model:
        return
    head = [r for r in rows if r["model"] == "piralix" and r["what"] == "decode" and r["batch"] == 1][0]
    emit({"metric": f"Piralix decode tok/s (B=1, {head['size']} layers, bf16 weights)", "value": head["tok_s"], "unit": "tok/s", "n_gpus": 1,
          "higher_is_better": True, "vs_baseline": None, "dtype": "bf16 weights, f32 residual, scores and state", "data": "synthetic", "rows": rows})
