"""Prefill and decode throughput of the Padulorn design (retention and windowed attention, a mixture of experts behind each) at
sizes that resemble a real model's layers, random weights, beside the closest existing model at equal size: Rivudra (windowed
attention beside a mixture of experts) with the same width, heads, key/value heads, window, layers, vocabulary, experts and
weights per expert, without a shared expert.

  python bench.py --model padulorn          (one JSON line)
  python tools/bench_padulorn.py [--only padulorn|rivudra] [--size 2048] [--case decode1,decode32,prefill1,prefill8]
"""
import argparse, os, sys

import torch

sys.path.insert(0, os.path.dirname(os.path.dirname(os.path.abspath(__file__))))
from tools.bench_gisitar import DECODE, DIM, LAYERS, PREFILL, VOCAB  # noqa: E402
from tools.bench_rivudra import init_experts, measure_rivudra, measure_routed  # noqa: E402

# width -> (heads of 128, key/value heads, window, kept first tokens, experts, top, groups, groups kept, expert ff)
SIZES = {1024: (8, 2, 1024, 16, 32, 4, 4, 2, 768), 2048: (16, 4, 1024, 16, 64, 4, 8, 4, 1536)}


def padulorn(width):
    from vyomai_amd import PadulornConfig, PadulornModel
    H, G, window, first, E, top, groups, keep, ff = SIZES[width]
    moe = {"kind": "moe", "router": {"experts": E, "top": top, "groups": {"count": groups, "keep": keep}}, "expert": {"ff": ff}}
    ret = {"type": "retention", "mixer": {"heads": H, "dim": DIM, "vdim": DIM, "rot": {"base": 10000.0, "dims": DIM},
                                          "decay": [1.0 - 2.0 ** -(5 + 7 * h / H) for h in range(H)]}, "mlp": moe}
    att = {"type": "attention", "mixer": {"heads": H, "kv_heads": G, "dim": DIM, "vdim": DIM, "scale": DIM ** -0.5, "v_mix": True,
                                          "mask": {"size": window, "keep_first": first},
                                          "rot": {"base": 10000.0, "dims": DIM, "scaling": {"factor": 4.0, "original": 4096, "fast": 32.0,
                                                                                            "slow": 1.0}}}, "mlp": moe}
    torch.manual_seed(0)
    with torch.device("cuda"):
        torch.set_default_dtype(torch.bfloat16)
        try:
            m = PadulornModel(PadulornConfig(vocab=VOCAB, width=width, layers=[att if i % 2 else ret for i in range(LAYERS)]))
        finally:
            torch.set_default_dtype(torch.float32)
    init_experts(m)
    return m.eval()


def measure_padulorn(width, cases):
    H, G, window, first, E, top, _, _, ff = SIZES[width]

    def cached(B, ctx):   # rings read, states read and written
        return LAYERS // 2 * B * (min(ctx, window + first) * G * 2 * DIM * 2 + 2 * H * DIM * DIM * 4)
    return measure_routed(padulorn(width), width, cases, E, top, 2 * width * ff, cached)


def rivudra(width, cases):
    H, G, window, _, E, top, groups, keep, ff = SIZES[width]
    return measure_rivudra(width, cases, (H, G, window, E, top, groups, keep, ff * 2 // 3, 0))


def run(sizes=tuple(SIZES), only=None, cases=None):
    cases = cases or list(PREFILL) + list(DECODE)
    out = {}
    for width in sizes:
        r = out[f"width {width}"] = {}
        for name, fn in (("padulorn", measure_padulorn), ("rivudra", rivudra)):
            if only in (None, name):
                r[name] = fn(width, cases)
                print(width, name, r[name], file=sys.stderr, flush=True)
                torch.cuda.empty_cache()
    return out


if __name__ == "__main__":
    ap = argparse.ArgumentParser()
    ap.add_argument("--only", choices=["padulorn", "rivudra"])
    ap.add_argument("--size", type=int, default=0)
    ap.add_argument("--case", default="")
    a = ap.parse_args()
    run((a.size,) if a.size else tuple(SIZES), a.only, a.case.split(",") if a.case else None)
