"""Prefill and decode throughput of the Gisitar design (latent + lightning attention) at sizes that resemble a real model's
layers, random weights, beside the closest existing model at equal size: the Gemma-style stack (pre-norm, gated MLP, one KV
head per query head, rotary positions) with the same width, heads, feed-forward and vocabulary.

  python bench.py --model gisitar          (one JSON line)
  python tools/bench_gisitar.py [--only gisitar|gemma] [--size 2048] [--case decode1,decode32,prefill1,prefill8]
"""
import argparse, os, sys, time, types

import torch
import torch.nn as nn

sys.path.insert(0, os.path.dirname(os.path.dirname(os.path.abspath(__file__))))

# width -> (heads of 128, q_rank, kv_rank, ff)
SIZES = {1024: (8, 512, 256, 4096), 2048: (16, 1024, 512, 8192)}
VOCAB, LAYERS, DIM = 32000, 8, 128
# name -> (batch, prompt tokens) of a prefill, (batch, context) of decode steps
PREFILL = {"prefill1": (1, 8192), "prefill8": (8, 1024)}
DECODE = {"decode1": (1, 4096), "decode32": (32, 2048)}


def gisitar(width):
    from vyomai_amd import GisitarConfig, GisitarModel
    H, qr, kr, ff = SIZES[width]
    lat = {"type": "latent_attention", "mixer": {"heads": H, "dim": DIM, "vdim": DIM, "q_rank": qr, "kv_rank": kr,
                                                 "scale": DIM ** -0.5}, "mlp": {"kind": "dense", "ff": ff}}
    lig = {"type": "lightning", "mixer": {"heads": H, "dim": DIM, "vdim": DIM,
                                          "decay": [2.718281828 ** -(2.0 ** -(1 + 6 * h / H)) for h in range(H)]},
           "mlp": {"kind": "dense", "ff": ff}}
    cfg = GisitarConfig(vocab=VOCAB, width=width, layers=[lig if i % 2 else lat for i in range(LAYERS)])
    torch.manual_seed(0)
    with torch.device("cuda"):
        torch.set_default_dtype(torch.bfloat16)
        try:
            m = GisitarModel(cfg)
        finally:
            torch.set_default_dtype(torch.float32)
    return m.eval()


class GemmaStack(nn.Module):
    """The language model of models/paligemma.py without its vision tower."""
    ROPE_OFFSET = 0

    def __init__(self, width, max_pos, heads, kv_heads, ff):
        super().__init__()
        from vyomai_amd.layers.positional_embeddings import RopeTable
        from vyomai_amd.models import paligemma as P
        t = types.SimpleNamespace(hidden_size=width, intermediate_size=ff, num_hidden_layers=LAYERS, num_attention_heads=heads,
                                  num_key_value_heads=kv_heads, head_dim=DIM, vocab_size=VOCAB, rms_norm_eps=1e-6,
                                  attention_bias=False, max_position_embeddings=max_pos, rope_theta=10000.0)
        self.shape = types.SimpleNamespace(text=t)
        self.embed_tokens = nn.Embedding(VOCAB, width)
        self.layers = nn.ModuleList([P.GemmaDecoderLayer(t, i) for i in range(LAYERS)])
        self.norm = P.GemmaRMSNorm(width)
        self.rope = RopeTable(P._angles(DIM, max_pos, 10000.0))

    def caches(self, B, cap):
        t = self.shape.text
        z = lambda: torch.zeros(B, t.num_key_value_heads, cap, DIM, dtype=torch.bfloat16, device="cuda")
        return [(z(), z()) for _ in self.layers]

    def prefill(self, ids, caches):
        from vyomai_amd import ops
        h = self.embed_tokens(ids)
        for layer, c in zip(self.layers, caches):
            h = layer(h, self.rope, 0, causal=True, cache=c)
        return ops.linear(self.norm(h[:, -1:]), self.embed_tokens.weight)


def timed(fn, iters, warm=2):
    for _ in range(warm):
        fn()
    s, e = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
    torch.cuda.synchronize()
    s.record()
    for _ in range(iters):
        fn()
    e.record()
    torch.cuda.synchronize()
    return s.elapsed_time(e) / iters


def measure_gisitar(width, cases):
    H, _, kr, _ = SIZES[width]
    m = gisitar(width)
    return measure_hybrid(m, width, cases, lambda B, ctx: B * sum(ctx * kr * 2 if l.mixer.kind == "latent" else 2 * H * DIM * DIM * 4
                                                                  for l in m.layers))


@torch.no_grad()
def measure_hybrid(m, width, cases, cached):
    """Throughputs of a hybrid decoder with dense feed-forwards; cached(B, context): bytes read and written per decode step besides
    the weights."""
    out = {"parameters": sum(p.numel() for p in m.parameters())}
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
            ms = timed(lambda: m.decode(ids, cache, slots), n - 5)
            nbytes = sum(p.numel() for p in m.parameters()) * 2 - VOCAB * width * 2 + cached(B, ctx)
            out[c] = {"batch": B, "context": ctx, "ms_per_step": round(ms, 4), "tokens_per_sec": round(B / ms * 1e3, 1),
                      "bytes_per_step": int(nbytes), "achieved_GBps": round(nbytes / ms * 1e-6, 1)}
        torch.cuda.empty_cache()
    return out


@torch.no_grad()
def measure_gemma(width, cases, heads=None, kv_heads=None, ff=None):
    from vyomai_amd.decode_plan import GemmaDecodePlan
    if heads is None:
        heads, _, _, ff = SIZES[width]
        kv_heads = heads
    torch.manual_seed(0)
    with torch.device("cuda"):
        m = GemmaStack(width, 8192 + 64, heads, kv_heads, ff)
    m = m.to(torch.bfloat16).eval()
    out = {"parameters": sum(p.numel() for p in m.parameters())}
    for c in cases:
        if c in PREFILL:
            B, L = PREFILL[c]
            ids = torch.randint(0, VOCAB, (B, L), device="cuda")
            caches = m.caches(B, L)
            ms = timed(lambda: m.prefill(ids, caches), 4)
            out[c] = {"batch": B, "prompt": L, "ms": round(ms, 3), "tokens_per_sec": round(B * L / ms * 1e3, 1)}
        else:
            B, ctx = DECODE[c]
            plan = GemmaDecodePlan(m, m.caches(B, ctx + 8), B)
            x = torch.randn(B, width, device="cuda", dtype=torch.bfloat16)
            ms = timed(lambda: plan.step(x, ctx - 1), 35)
            nbytes = sum(p.numel() for p in m.parameters()) * 2 + B * LAYERS * ctx * 2 * kv_heads * DIM * 2
            out[c] = {"batch": B, "context": ctx, "ms_per_step": round(ms, 4), "tokens_per_sec": round(B / ms * 1e3, 1),
                      "bytes_per_step": int(nbytes), "achieved_GBps": round(nbytes / ms * 1e-6, 1)}
            del plan
        torch.cuda.empty_cache()
    return out


def run(sizes=tuple(SIZES), only=None, cases=None):
    cases = cases or list(PREFILL) + list(DECODE)
    out = {}
    for width in sizes:
        r = out[f"width {width}"] = {}
        for name, fn in (("gisitar", measure_gisitar), ("gemma", measure_gemma)):
            if only in (None, name):
                r[name] = fn(width, cases)
                print(width, name, r[name], file=sys.stderr, flush=True)
                torch.cuda.empty_cache()
    return out


if __name__ == "__main__":
    ap = argparse.ArgumentParser()
    ap.add_argument("--only", choices=["gisitar", "gemma"])
    ap.add_argument("--size", type=int, default=0)
    ap.add_argument("--case", default="")
    a = ap.parse_args()
    run((a.size,) if a.size else tuple(SIZES), a.only, a.case.split(",") if a.case else None)
