"""Prefill and decode throughput of the Biruvik design (gated linear attention, differential attention, windowed latent attention) at
sizes that resemble a real model's layers, random weights, beside the closest existing model at equal size: Gisitar (lightning and
latent attention, norms on both sides of every sublayer too) with the same width, heads, latents, layers, vocabulary and weights per
feed-forward.

  python bench.py --model biruvik          (one JSON line)
  python tools/bench_biruvik.py [--only biruvik|gisitar] [--size 2048] [--case decode1,decode32,prefill1,prefill8]
"""
import argparse, os, sys

import torch

sys.path.insert(0, os.path.dirname(os.path.dirname(os.path.abspath(__file__))))
from tools import bench_gisitar  # noqa: E402
from tools.bench_gisitar import DECODE, DIM, LAYERS, PREFILL, VOCAB, measure_gisitar, measure_hybrid  # noqa: E402

# width -> (heads of 128, key/value heads of the differential layers, window and kv_rank of the latent ones, ff)
SIZES = {w: (H, H // 4, 1024, kr, ff * 3 // 2) for w, (H, _, kr, ff) in bench_gisitar.SIZES.items()}
ORDER = ("hgrn2", "attention", "hgrn2", "latent_attention")


def biruvik(width):
    from vyomai_amd import BiruvikConfig, BiruvikModel
    H, G, window, kr, ff = SIZES[width]
    mixers = {"hgrn2": {"heads": H, "dim": DIM, "vdim": DIM},
              "attention": {"heads": H, "kv_heads": G, "dim": DIM // 2, "vdim": DIM, "scale": (DIM // 2) ** -0.5, "diff": 0.5,
                            "q_temp": {"coef": 0.1, "every": 4096}},
              "latent_attention": {"heads": H, "dim": DIM, "vdim": DIM, "kv_rank": kr, "scale": DIM ** -0.5, "mask": {"size": window}}}
    layers = [{"type": k, "mixer": mixers[k], "mlp": {"kind": "dense", "ff": ff}} for k in (ORDER * LAYERS)[:LAYERS]]
    torch.manual_seed(0)
    with torch.device("cuda"):
        torch.set_default_dtype(torch.bfloat16)
        try:
            m = BiruvikModel(BiruvikConfig(vocab=VOCAB, width=width, layers=layers, logit_softcap=30.0))
        finally:
            torch.set_default_dtype(torch.float32)
    return m.eval()


def measure_biruvik(width, cases):
    H, G, window, kr, _ = SIZES[width]
    m = biruvik(width)

    def cached(B, ctx):   # rows read, states read and written
        per = {"gated": 2 * H * DIM * DIM * 4, "differential": ctx * G * 2 * DIM * 2, "latent": min(ctx, window) * kr * 2}
        return B * sum(per[l.mixer.kind] for l in m.layers)
    return measure_hybrid(m, width, cases, cached)


def run(sizes=tuple(SIZES), only=None, cases=None):
    cases = cases or list(PREFILL) + list(DECODE)
    out = {}
    for width in sizes:
        r = out[f"width {width}"] = {}
        for name, fn in (("biruvik", measure_biruvik), ("gisitar", measure_gisitar)):
            if only in (None, name):
                r[name] = fn(width, cases)
                print(width, name, r[name], file=sys.stderr, flush=True)
                torch.cuda.empty_cache()
    return out


if __name__ == "__main__":
    ap = argparse.ArgumentParser()
    ap.add_argument("--only", choices=["biruvik", "gisitar"])
    ap.add_argument("--size", type=int, default=0)
    ap.add_argument("--case", default="")
    a = ap.parse_args()
    run((a.size,) if a.size else tuple(SIZES), a.only, a.case.split(",") if a.case else None)
