"""Prefill and decode throughput of the Rivudra design (windowed attention beside a mixture of experts) at sizes that resemble a
real model's layers, random weights, beside the closest existing model at equal size: the Gemma-style stack (pre-norm, gated
MLP, rotary positions) with the same width, heads, key/value heads, layers and vocabulary, and a feed-forward as wide as what
one token of the design goes through (top experts + the shared one).

  python bench.py --model rivudra          (one JSON line)
  python tools/bench_rivudra.py [--only rivudra|gemma] [--size 2048] [--case decode1,decode32,prefill1,prefill8]
"""
import argparse, os, sys

import torch

sys.path.insert(0, os.path.dirname(os.path.dirname(os.path.abspath(__file__))))
from tools.bench_gisitar import DECODE, DIM, LAYERS, PREFILL, VOCAB, measure_gemma, timed  # noqa: E402

# width -> (heads of 128, key/value heads, window, experts, top, groups, groups kept, expert ff, shared ff)
SIZES = {1024: (8, 2, 1024, 32, 4, 4, 2, 512, 1024), 2048: (16, 4, 1024, 64, 4, 8, 4, 1024, 2048)}


def init_experts(m):
    with torch.no_grad():
        for l in m.layers:
            for p in (l.mlp.gate, l.mlp.up, l.mlp.down):
                if p is not None:
                    p.normal_(std=p.shape[-1] ** -0.5)


def rivudra(width, size=None):
    from vyomai_amd import RivudraConfig, RivudraModel
    H, G, window, E, top, groups, keep, ff, shared = size or SIZES[width]
    layer = {"type": "attention", "mixer": {"heads": H, "kv_heads": G, "dim": DIM, "vdim": DIM, "scale": DIM ** -0.5,
                                            "mask": {"size": window}, "rot": {"base": 10000.0, "dims": DIM}},
             "mlp": {"kind": "moe", "router": {"experts": E, "top": top, "scale": 1.0, "groups": {"count": groups, "keep": keep}},
                     "expert": {"ff": ff, "limit": 7.0}, "shared": {"ff": shared, "limit": 7.0} if shared else None}}
    torch.manual_seed(0)
    with torch.device("cuda"):
        torch.set_default_dtype(torch.bfloat16)
        try:
            m = RivudraModel(RivudraConfig(vocab=VOCAB, width=width, layers=[layer] * LAYERS))
        finally:
            torch.set_default_dtype(torch.float32)
    init_experts(m)
    return m.eval()


def measure_rivudra(width, cases, size=None):
    H, G, window, E, top, _, _, ff, _ = size or SIZES[width]

    def cached(B, ctx):
        return LAYERS * B * min(ctx, window) * G * 2 * DIM * 2
    return measure_routed(rivudra(width, size), width, cases, E, top, 3 * width * ff, cached)


@torch.no_grad()
def measure_routed(m, width, cases, E, top, expert, cached):
    """Throughputs of a hybrid decoder whose layers all have a mixture: `expert` weights per expert, cached(B, context) bytes read
    per decode step besides weights."""
    total = sum(p.numel() for p in m.parameters())
    out = {"parameters": total, "active_parameters": total - LAYERS * (E - top) * expert}
    for c in cases:
        if c in PREFILL:
            B, L = PREFILL[c]
            ids = torch.randint(0, VOCAB, (B, L), device="cuda")
            cache = m.new_cache(B, L)

            def go():
                slots = cache.allocate(B)
                x = m.prefill(ids, [L] * B, cache, slots)
                m.logits(x[:, -1])
                cache.free(slots)
            ms = timed(go, 4)
            out[c] = {"batch": B, "prompt": L, "ms": round(ms, 3), "tokens_per_sec": round(B * L / ms * 1e3, 1)}
        else:
            B, ctx = DECODE[c]
            n = 40
            cache = m.new_cache(B, ctx + n + 8)
            slots = cache.allocate(B)
            cache.advance(slots, [ctx - n // 2] * B)          # a context of zeros: the kernels' work does not depend on it
            ids = torch.randint(0, VOCAB, (B,), device="cuda")
            # experts in use per layer of this batch (the routers' own choice)
            h = torch.randn(B, width, device="cuda", dtype=torch.bfloat16)
            used = sum(int(l.mlp.routed(h).ids.unique().numel()) for l in m.layers)
            ms = timed(lambda: m.decode(ids, cache, slots), n - 5)
            nbytes = (total - VOCAB * width - LAYERS * E * expert + used * expert) * 2 + cached(B, ctx)
            out[c] = {"batch": B, "context": ctx, "ms_per_step": round(ms, 4), "tokens_per_sec": round(B / ms * 1e3, 1),
                      "experts_per_layer": round(used / LAYERS, 1), "bytes_per_step": int(nbytes),
                      "achieved_GBps": round(nbytes / ms * 1e-6, 1)}
        torch.cuda.empty_cache()
    return out


def gemma(width, cases):
    H, G, _, _, top, _, _, ff, shared = SIZES[width]
    return measure_gemma(width, cases, H, G, top * ff + shared)


def run(sizes=tuple(SIZES), only=None, cases=None):
    cases = cases or list(PREFILL) + list(DECODE)
    out = {}
    for width in sizes:
        r = out[f"width {width}"] = {}
        for name, fn in (("rivudra", measure_rivudra), ("gemma", gemma)):
            if only in (None, name):
                r[name] = fn(width, cases)
                print(width, name, r[name], file=sys.stderr, flush=True)
                torch.cuda.empty_cache()
    return out


if __name__ == "__main__":
    ap = argparse.ArgumentParser()
    ap.add_argument("--only", choices=["rivudra", "gemma"])
    ap.add_argument("--size", type=int, default=0)
    ap.add_argument("--case", default="")
    a = ap.parse_args()
    run((a.size,) if a.size else tuple(SIZES), a.only, a.case.split(",") if a.case else None)
