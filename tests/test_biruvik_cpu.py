"""Biruvik without a GPU: the oracle against closed forms, checkpoint loading, packing, the cache's bookkeeping, and argument checks
of the C ABI."""
import ctypes
import math

import pytest
import torch

from oracle import biruvik_oracle as O
from tests import biruvik_cases as P


def rand(*shape, seed=0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed), dtype=torch.float64)


# ---- the oracle -----------------------------------------------------------------------------------
@pytest.mark.parametrize("size", [None, 1, 4, 20])
def test_oracle_attention_is_the_masked_softmax(size):
    T = 11
    q, k, v = rand(T, 3, seed=1), rand(T, 3, seed=2), rand(T, 5, seed=3)
    i, j = torch.arange(T)[:, None], torch.arange(T)[None]
    hidden = (j > i) | (i - j >= (size or T))
    want = (q @ k.T * 0.7).masked_fill(hidden, float("-inf")).softmax(-1) @ v
    assert torch.allclose(O.softmax_attention(q, k, v, 0.7, size), want)


def test_oracle_temperature():
    t = [O.temperature(p, 0.5, 4) for p in range(13)]
    assert t[:3] == [1.0] * 3 and t[3:7] == [1 + 0.5 * math.log(2)] * 4 and t[11] == 1 + 0.5 * math.log(4) and t[12] == t[11]
    assert O.temperature(5, 0.0, 1) == 1.0 and O.temperature(0, 1.0, 1) == 1 + math.log(2)


def test_oracle_difference():
    p = {"lq1": torch.tensor([1.0, 2.0]), "lk1": torch.tensor([0.5, -0.25]), "lq2": torch.tensor([1.0, 0.0]), "lk2": torch.tensor([0.5, 9.0])}
    assert abs(float(O.difference_weight(p, 0.4)) - (1.0 - math.exp(0.5) + 0.4)) < 1e-6
    a1, a2 = rand(3, 6, seed=1), rand(3, 6, seed=2)
    y = O.differential_head(a1, a2, torch.tensor(0.7), 0.25, 0.0)
    d = a1 - 0.7 * a2
    assert torch.allclose(y.pow(2).mean(-1).sqrt(), torch.full((3,), 0.75, dtype=torch.float64))
    assert torch.allclose(torch.nn.functional.cosine_similarity(y, d, dim=-1), torch.ones(3, dtype=torch.float64))
    assert torch.equal(O.differential_head(a1, a2, torch.tensor(0.0), 0.0, 1.0), O.rms(a1, 1.0))


def test_oracle_recurrence_is_gated_attention():
    T = 9
    q, v = rand(T, 4, seed=1), rand(T, 3, seed=3)
    f = torch.sigmoid(rand(T, 4, seed=2) + 1)
    g = torch.cumsum(torch.log(f), 0)                       # the gates between two tokens: differences of sums of logarithms
    A = torch.zeros(T, T, dtype=torch.float64)
    for i in range(T):
        for j in range(i + 1):
            A[i, j] = (q[i] * (1 - f[j]) * torch.exp(g[i] - g[j])).sum()
    assert torch.allclose(O.recurrence(q, f, v), A @ v)
    S = torch.zeros(4, 3, dtype=torch.float64)
    parts = torch.cat([O.recurrence(q[a:b], f[a:b], v[a:b], S) for a, b in ((0, 2), (2, 3), (3, 9))])
    assert torch.allclose(parts, A @ v)


def test_oracle_gates_and_small_functions():
    z, lower = torch.tensor([-50.0, 0.0, 50.0]).double(), torch.tensor([0.25, 0.5, 0.0]).double()
    assert torch.allclose(O.forget(z, lower), torch.tensor([0.25, 0.75, 1.0]).double())
    assert torch.equal(O.mlp(torch.tensor([[2.0, -3.0]]), {"up": torch.eye(2), "down": torch.eye(2)}), torch.tensor([[4.0, 0.0]]))
    x = torch.tensor([0.01, 3.0, 1e4]).double()
    assert torch.allclose(O.softcap(x, 5.0), torch.tensor([0.01 - 0.01 ** 3 / 75, 5 * math.tanh(0.6), 5.0]).double())
    assert torch.allclose(O.rms(torch.tensor([[3.0, 4.0]]), 0.0), torch.tensor([[0.6, 0.8]]) * 2 ** 0.5)


@pytest.mark.parametrize("name", list(P.CONFIGS))
def test_oracle_is_causal(name):
    cfg, w = P.CONFIGS[name], P.weights(P.CONFIGS[name])
    ids = P.tokens(cfg, 8)
    full = O.forward(w, cfg, ids)
    assert torch.allclose(full[:5], O.forward(w, cfg, ids[:5]), atol=1e-12) and full.abs().max() <= cfg["logit_softcap"]


# ---- loading and packing --------------------------------------------------------------------------
@pytest.mark.parametrize("name", list(P.CONFIGS))
def test_checkpoint_loads_by_name(name, tmp_path):
    from vyomai_amd import BiruvikModel, load_pretrained
    cfg, w = P.CONFIGS[name], P.weights(P.CONFIGS[name])
    P.write_folder(tmp_path, cfg, w)
    m = load_pretrained(str(tmp_path), torch.float32, "cpu")
    assert isinstance(m, BiruvikModel) and m.softcap == cfg["logit_softcap"] and m.embed_scale == cfg["embedding"]["scale"]
    seen = set()
    for n, p in m.named_parameters():
        k = m.checkpoint_name(n)
        assert torch.equal(p, w[k]), k
        seen.add(k)
    assert seen == set(w)


def test_checkpoint_and_configuration_errors(tmp_path):
    from vyomai_amd import load_pretrained
    cfg, w = P.CONFIGS["edges"], P.weights(P.CONFIGS["edges"])
    P.write_folder(tmp_path, cfg, {n: t for n, t in w.items() if n != "l0.mix.k.b"})
    with pytest.raises(KeyError, match="l0.mix.k.b"):
        load_pretrained(str(tmp_path), torch.float32, "cpu")
    P.write_folder(tmp_path, cfg, {**w, "l1.mix.dq": w["l1.mix.q"]})
    with pytest.raises(KeyError, match="l1.mix.dq"):
        load_pretrained(str(tmp_path), torch.float32, "cpu")
    for change, match in (({"type": "sieve"}, "sieve"), ({"mlp": {"kind": "sieve"}}, "sieve")):
        P.write_folder(tmp_path, {**cfg, "layers": [{**cfg["layers"][0], **change}]}, w)
        with pytest.raises(ValueError, match=match):
            load_pretrained(str(tmp_path), torch.float32, "cpu")


def test_impossible_sizes_are_refused():
    from vyomai_amd.layers.differential_attention import DifferentialAttention
    from vyomai_amd.layers.ffn import PlainFeedForward
    from vyomai_amd.layers.gated_linear_attention import GatedLinearAttention
    from vyomai_amd.layers.latent_attention import LatentAttention
    from vyomai_amd.models.hybrid import HybridDecoderModel, ParallelLayer
    with pytest.raises(ValueError, match="query heads"):
        DifferentialAttention(8, 3, 2, 8, 8, 1.0, 0.5, 1e-5)
    with pytest.raises(ValueError, match="scale"):
        DifferentialAttention(8, 2, 2, 8, 8, 0.0, 0.5, 1e-5)
    with pytest.raises(ValueError, match="every 2.5"):
        DifferentialAttention(8, 2, 2, 8, 8, 1.0, 0.5, 1e-5, 0.1, 2.5)
    with pytest.raises(ValueError, match="window"):
        LatentAttention(8, 1, 8, 8, None, 8, 1.0, 1e-5, window=0)
    with pytest.raises(ValueError, match="capped"):
        HybridDecoderModel(None, 8, 8, [], 1e-5, "rms", softcap=-1.0)
    with pytest.raises(ValueError, match="parallel"):
        ParallelLayer(8, GatedLinearAttention(8, 1, 8, 8, 1e-5), PlainFeedForward(8, 8), 1e-5).packed()
    with pytest.raises(ValueError, match="biases"):
        ParallelLayer(8, DifferentialAttention(8, 2, 2, 8, 8, 1.0, 0.5, 1e-5), None, 1e-5).packed()


@pytest.mark.parametrize("name", list(P.CONFIGS))
def test_packed_products_are_the_separate_ones(name, tmp_path):
    from vyomai_amd import load_pretrained
    from vyomai_amd.ops import up8
    cfg, w = P.CONFIGS[name], P.weights(P.CONFIGS[name])
    P.write_folder(tmp_path, cfg, w)
    m = load_pretrained(str(tmp_path), torch.float32, "cpu")
    W = cfg["width"]
    x = rand(W, seed=3).float()
    xp = torch.zeros(up8(W))
    xp[:W] = x

    def heads(rows, n, dim):
        r = rows.view(n, up8(dim))
        assert not r[:, dim:].any()
        return r[:, :dim].reshape(-1)

    for i, l in enumerate(cfg["layers"]):
        mix, mod, pre = l["mixer"], m.layers[i].mixer, f"l{i}."
        p = mod.packed()
        H, dk, dv = mix["heads"], mix["dim"], mix["vdim"]
        rows, at = p.w_in @ xp + (getattr(p, "b_in", None) if hasattr(p, "b_in") else 0.0), 0
        parts = {"attention": lambda: (("q", 2 * H, dk), ("k", 2 * mix["kv_heads"], dk), ("v", mix["kv_heads"], dv)),
                 "latent_attention": lambda: (("q", H, dk), ("dkv", 1, mix["kv_rank"]), ("g", 1, H)),
                 "hgrn2": lambda: (("q", H, dk), ("f", H, dk), ("v", H, dv))}[l["type"]]()
        for n, count, dim in parts:
            want = w[pre + "mix." + n] @ x
            if l["type"] == "attention":
                want = want + w[f"{pre}mix.{n}.b"]
            assert torch.allclose(heads(rows[at: at + count * up8(dim)], count, dim), want, atol=1e-4), n
            at += count * up8(dim)
        assert at == rows.numel()
        o, op = rand(H, dv, seed=4).float(), torch.zeros(H, up8(dv))
        op[:, :dv] = o
        y = p.w_o @ op.view(-1)
        assert torch.allclose(y[:W], w[pre + "mix.o"] @ o.view(-1), atol=1e-4) and not y[W:].any()
        n = m.layers[i].packed()
        for k in ("norm1", "norm1b") + (("norm2", "norm2b") if l["mlp"] is not None else ()):
            v = getattr(n, k)
            assert torch.equal(v[:W], w[pre + k].expand(W)) and not v[W:].any()          # one number, everywhere but in the padding
        if l["type"] == "attention":
            c = mod.constants()
            assert (c.prep.n_q, c.prep.group, c.prep.temp_every) == (dk, up8(dk), mix["q_temp"]["every"])
            assert torch.equal(heads(c.prep.q_norm, 2 * H, dk), w[pre + "mix.q.norm"].repeat(2 * H))
            assert torch.equal(heads(c.prep.k_norm, 2 * mix["kv_heads"], dk), w[pre + "mix.k.norm"].repeat(2 * mix["kv_heads"]))
            lam = O.difference_weight({k: w[f"{pre}mix.{k}"].double() for k in ("lq1", "lk1", "lq2", "lk2")}, mix["diff"])
            assert abs(c.diff.lambda_ - float(lam)) < 1e-6 and abs(c.diff.out_scale - (1 - mix["diff"])) < 1e-6 and c.diff.n_v == dv
        if l["type"] == "hgrn2":
            assert torch.equal(heads(p.f_bias, H, dk), w[pre + "mix.f.b"])
            low = p.f_lower.view(H, up8(dk))
            assert torch.allclose(low[:, :dk].reshape(-1), w[pre + "mix.lower"], atol=1e-7) and bool((low[:, dk:] == 1).all())
        if l["mlp"] is not None:
            q, ff = m.layers[i].mlp.packed(), l["mlp"]["ff"]
            up = q.w_up @ xp
            assert torch.allclose(up[:ff], w[pre + "mlp.up"] @ x, atol=1e-4) and not up[ff:].any()
    assert torch.equal(m.packed().final_norm[:W], w["final.norm"].expand(W))


def test_cache_bookkeeping():
    """A windowed latent is a ring of one head; differential rows never wrap and grow with the sequences."""
    from vyomai_amd import SlotCache
    from vyomai_amd.layers.differential_attention import DifferentialAttention
    from vyomai_amd.layers.latent_attention import LatentAttention
    specs = [LatentAttention(8, 2, 8, 8, None, 13, 1.0, 1e-5, window=9, head_gate=True).cache_spec(),
             DifferentialAttention(8, 4, 2, 5, 11, 1.0, 0.5, 1e-5).cache_spec(), LatentAttention(8, 2, 8, 8, 8, 13, 1.0, 1e-5).cache_spec()]
    c = SlotCache(specs, torch.float32, "cpu", slots=1, capacity=4)
    assert [tuple(b.shape) for b in c.buffers] == [(1, 1, 4, 16), (1, 2, 4, 32), (1, 4, 16)]
    [a] = c.allocate(1)
    c.reserve([a], [3])
    c.advance([a], [3])
    for b in c.buffers:
        b[a, ..., :3, :] = torch.arange(3.0)[:, None]
    c.reserve([a], [30])
    assert [b.shape[-2] for b in c.buffers] == [9, 33, 33]
    for b in c.buffers:
        assert torch.equal(b[a, ..., :3, 0].reshape(-1, 3)[-1], torch.arange(3.0)) and not b[a, ..., 3:, :].any()
    c.reserve([a], [500])
    assert [b.shape[-2] for b in c.buffers] == [9, c.capacity, c.capacity]


def test_argument_errors_without_a_gpu():
    from vyomai_amd import _lib
    buf = (ctypes.c_char * 4096)()
    p = (ctypes.addressof(buf) + 63) // 64 * 64
    ref = ctypes.byref

    def fails(match, name, *args):
        with pytest.raises(_lib.VyomHipError, match=match):
            _lib.call(name, *args)
    for kw, match in (({"group": 5, "n": 5}, "norms over"), ({"group": 8, "n": 9}, "norms over"), ({"group": 8, "n": 8, "every": -1}, "norms over"),
                      ({"group": 0, "n": 8, "every": 4}, "temperature")):
        prep = _lib.VyQkvPrep(p, p, kw["n"], kw["n"], 1e-5, 0.0, group=kw["group"], temp_every=kw.get("every", 0))
        fails(match, "vy_qkv_rows", p, 64, 0, 16, 32, ref(prep), p, 96, 96, 4, 0, None, 0, 0, 1, None, p, None, 1, 1, 1, 1, 16, 8, 1, None)
    prep, diff = _lib.VyQkvPrep(p, p, 8, 8, 1e-5, 0.0, group=8), _lib.VyDiff(0.5, 0.5, 1e-5, 8)

    def decode(prep=prep, diff=diff, keep=0, og=-1, sink=0, top=1, dim=16):
        return ["vy_window_decode", p, 64, 0, 16, 32, og, p, 96, 96, 4, keep, None, 0, 0, ref(prep) if prep else None, ref(diff), None, p, top, p, 8,
                1, 1, 1, dim, 8, 1.0, sink, None, 0, 1, None]
    for kw in ({"prep": None}, {"keep": 1}, {"og": 40}, {"sink": 1}, {"top": 5}, {"diff": _lib.VyDiff(0.5, 0.5, 1e-5, 9)}, {"dim": 8}):
        fails("bad differential attention|norms over", *decode(**kw))
    fails("workspace", *decode())

    def attn(R=4, L=2, dim=16, n_v=8, ldq=16, r_sh=96):
        return ["vy_diff_attn_fwd", p, ldq, p, 96, r_sh, R, ref(_lib.VyDiff(0.5, 0.5, 1e-5, n_v)), None, p, None, p, 8, 1, L, 1, 1, dim, 8, 1.0, 1, None]
    for kw, match in (({"L": 5}, "bad arguments"), ({"dim": 24}, "multiples of 8"), ({"ldq": 8}, "multiples of 8"), ({"R": 5}, "ring strides"),
                      ({"n_v": 0}, "norm over")):
        fails(match, *attn(**kw))
    fails("workspace", "vy_gated_attn", p, 24, 0, 8, 16, p, p, p, None, p, None, p, 8, 1, 2, 1, 8, 8, 1, None, 0, 1, None)
    fails("multiples of 8", "vy_gated_attn", p, 24, 0, 4, 16, p, p, p, None, p, None, p, 8, 1, 1, 1, 8, 8, 1, None, 0, 1, None)
    fails("null", "vy_gated_attn", p, 24, 0, 8, 16, p, p, None, None, p, None, p, 8, 1, 1, 1, 8, 8, 1, None, 0, 1, None)
    fails("512", "vy_gated_attn", p, 2000, 0, 520, 1040, p, p, p, None, p, None, p, 8, 1, 1, 1, 520, 8, 1, None, 0, 0, None)
    fails("cap", "vy_linear_softcap_fwd", p, 8, p, 8, p, 8, 1, 8, 8, 0.0, 1, None)
    fails("unknown activation", "vy_linear_fwd", p, 8, p, 8, None, None, 0, p, 8, None, 1, 8, 8, 5, 1, None)
    fails("bad arguments", "vy_latent_norm", p, 16, None, None, 0, 8, -8, p, None, 0, 8, 8, None, 0, 0, 0, 0, None, None, None, 1, 1, 1e-5, 1, None)
    fails("empty", "vy_latent_decode", p, 8, p, p, p, 8, 8, None, p, 1, p, 8, None, 0, 0, -1, 1, 1, 8, 8, 8, 1.0, p, 4096, 1, None)
