"""Padulorn without a GPU: the oracle against closed forms, checkpoint loading, packing, rotary tables, the ring's bookkeeping, and
argument checks of the C ABI."""
import ctypes
import math

import pytest
import torch

from oracle import padulorn_oracle as O
from tests import padulorn_cases as P


def rand(*shape, seed=0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed), dtype=torch.float64)


# ---- the oracle -----------------------------------------------------------------------------------
@pytest.mark.parametrize("size,first", [(4, 0), (4, 2), (1, 3), (20, 1), (2, 20)])
def test_oracle_window_attention_is_the_masked_softmax(size, first):
    T = 11
    q, k, v = rand(T, 3, seed=1), rand(T, 3, seed=2), rand(T, 5, seed=3)
    i, j = torch.arange(T)[:, None], torch.arange(T)[None]
    hidden = (j > i) | ((i - j >= size) & (j >= first))
    want = (q @ k.T * 0.7).masked_fill(hidden, float("-inf")).softmax(-1) @ v
    assert torch.allclose(O.window_attention(q, k, v, 0.7, size, first), want)


@pytest.mark.parametrize("layout", ["pairs", "halves"])
def test_oracle_rotation(layout):
    q, k = rand(1, 10, seed=2), rand(1, 10, seed=3)
    rot = {"base": 50.0, "dims": 6}
    a = O.rotate(q, rot, layout, 11)
    assert torch.allclose(a.norm(), q.norm()) and torch.equal(a[:, 6:], q[:, 6:]) and not torch.allclose(a[:, :6], q[:, :6])
    assert torch.allclose(O.rotate(q, rot, layout, 0), q)
    dot = [(O.rotate(q, rot, layout, p + 3) * O.rotate(k, rot, layout, p)).sum() for p in (0, 5, 40)]
    assert torch.allclose(dot[0], dot[1]) and torch.allclose(dot[0], dot[2])
    # a complex number of the two columns of a pair turns
    one = (2, 3) if layout == "pairs" else (1, 4)
    z, y = torch.complex(q[0, one[0]], q[0, one[1]]), torch.complex(a[0, one[0]], a[0, one[1]])
    angle = torch.tensor(11 * 50.0 ** (-2 / 6), dtype=torch.float64)
    assert torch.allclose(y, z * torch.polar(torch.ones_like(angle), angle))


def test_oracle_frequencies():
    rot = {"base": 100.0, "dims": 12}
    f, c = O.frequencies(rot)
    assert c == 1.0 and f[0] == 1.0 and abs(f[3] - 0.1) < 1e-15
    g, c = O.frequencies({**rot, "scaling": P.yarn(8.0, 60, 5.0, 0.7)})
    assert abs(c - (1 + 0.1 * math.log(8.0))) < 1e-15
    assert g[0] == f[0] and abs(g[5] - f[5] / 8.0) < 1e-15           # many turns: kept; hardly any: divided
    ratio = [b / a for a, b in zip(f, g)]
    assert all(x >= y - 1e-15 for x, y in zip(ratio, ratio[1:])) and any(0.126 < r < 0.999 for r in ratio)
    g, _ = O.frequencies({**rot, "scaling": P.yarn(8.0, 60, 2.0, 2.0)})   # an (all but) empty ramp: a step
    assert sorted(set(round(b / a, 12) for a, b in zip(f, g))) in ([0.125, 1.0], [1.0])


def test_oracle_recurrence_is_decayed_attention():
    T = 9
    q, k, v = rand(T, 4, seed=1), rand(T, 4, seed=2), rand(T, 3, seed=3)
    i, j = torch.arange(T)[:, None], torch.arange(T)[None]
    want = (q @ k.T * torch.where(j <= i, 0.8 ** (i - j).double(), torch.zeros(()))) @ v
    assert torch.allclose(O.recurrence(q, k, v, 0.8), want)
    S = torch.zeros(4, 3, dtype=torch.float64)
    parts = torch.cat([O.recurrence(q[a:b], k[a:b], v[a:b], 0.8, S) for a, b in ((0, 2), (2, 3), (3, 9))])
    assert torch.allclose(parts, want)


def test_oracle_routing():
    cfg = {"experts": 6, "top": 2, "groups": {"count": 3, "keep": 1}}
    z = torch.tensor([-3.0, 3.0, 1.9, 1.8, 1.0, 2.0], dtype=torch.float64)     # groups (0, 1), (2, 3), (4, 5)
    chosen, w = O.route(z, cfg)                       # the best pair, not the best expert, makes the best group
    assert chosen == [2, 3] and abs(w[0] - 1 / (1 + math.exp(-1.9))) < 1e-12
    cfg["groups"]["keep"] = 2
    assert O.route(z, cfg)[0] == [5, 2]
    cfg["groups"]["keep"] = 3
    assert O.route(z, cfg)[0] == [1, 5]
    cfg["groups"] = {"count": 6, "keep": 2}           # groups of one
    assert O.route(z, cfg)[0] == [1, 5]


@pytest.mark.parametrize("name", list(P.CONFIGS))
def test_oracle_is_causal(name):
    cfg, w = P.CONFIGS[name], P.weights(P.CONFIGS[name])
    ids = P.tokens(cfg, 8)
    full = O.forward(w, cfg, ids)
    assert torch.allclose(full[:5], O.forward(w, cfg, ids[:5]), atol=1e-12)


# ---- loading and packing --------------------------------------------------------------------------
@pytest.mark.parametrize("name", list(P.CONFIGS))
def test_checkpoint_loads_by_name(name, tmp_path):
    from vyomai_amd import PadulornModel, load_pretrained
    cfg, w = P.CONFIGS[name], P.weights(P.CONFIGS[name])
    P.write_folder(tmp_path, cfg, w)
    m = load_pretrained(str(tmp_path), torch.float32, "cpu")
    assert isinstance(m, PadulornModel)

    def check():
        seen = set()
        for n, p in m.named_parameters():
            keys = m.checkpoint_name(n)
            for i, k in enumerate(keys if isinstance(keys, list) else [keys]):
                assert torch.equal(p[i] if isinstance(keys, list) else p, w[k]), k
                seen.add(k)
        assert seen == set(w)
    check()
    for l in m.layers:                       # packed experts are views of one storage and still hold the same values
        if l.mlp is not None:
            p = l.mlp.packed()
            assert l.mlp.up.untyped_storage().data_ptr() == p.w_gu.untyped_storage().data_ptr() and l.mlp.packed() is p
    check()
    from vyomai_amd.layers.window_attention import VALUES_FIRST, VALUES_MIX, VALUES_OWN
    first = True
    for l, spec in zip(m.layers, cfg["layers"]):
        if spec["type"] == "attention":
            mixes = spec["mixer"]["v_mix"]
            assert l.mixer.values == (VALUES_OWN if not mixes else VALUES_FIRST if first else VALUES_MIX)
            first = first and not mixes


def test_checkpoint_and_configuration_errors(tmp_path):
    from vyomai_amd import load_pretrained
    cfg, w = P.CONFIGS["edges"], P.weights(P.CONFIGS["edges"])
    P.write_folder(tmp_path, cfg, {n: t for n, t in w.items() if n != "l2.mix.vmix"})
    with pytest.raises(KeyError, match="l2.mix.vmix"):
        load_pretrained(str(tmp_path), torch.float32, "cpu")
    P.write_folder(tmp_path, cfg, {**w, "l1.mix.q.norm": w["l0.mix.q.norm"]})      # a norm that the layer does not have
    with pytest.raises(KeyError, match="l1.mix.q.norm"):
        load_pretrained(str(tmp_path), torch.float32, "cpu")
    for change, match in (({"type": "sieve"}, "sieve"), ({"mlp": {"kind": "sieve"}}, "sieve")):
        P.write_folder(tmp_path, {**cfg, "layers": [{**cfg["layers"][0], **change}]}, w)
        with pytest.raises(ValueError, match=match):
            load_pretrained(str(tmp_path), torch.float32, "cpu")


def test_impossible_sizes_are_refused():
    from vyomai_amd.layers.ffn import MixtureFeedForward
    from vyomai_amd.layers.retention import Retention
    from vyomai_amd.layers.window_attention import WindowAttention
    for kw in ({"act": "relu"}, {"score": "tanh"}, {"group_best": 3}):
        with pytest.raises(ValueError):
            MixtureFeedForward(8, 4, 1, 8, **kw)
    with pytest.raises(ValueError, match="kept"):
        WindowAttention(8, 2, 1, 8, 8, 1.0, 4, keep_first=-1)
    with pytest.raises(ValueError, match="decays"):
        Retention(8, 2, 8, 8, [0.5], 1e-5)
    with pytest.raises(ValueError, match="rotated"):
        Retention(8, 2, 8, 8, [0.5, 0.5], 1e-5, rot_dims=10)


@pytest.mark.parametrize("name", list(P.CONFIGS))
def test_packed_products_are_the_separate_ones(name, tmp_path):
    from vyomai_amd import load_pretrained, ops
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
        mix, p, pre, mod = l["mixer"], m.layers[i].mixer.packed(), f"l{i}.", m.layers[i]
        H, dk, dv = mix["heads"], mix["dim"], mix["vdim"]
        G = mix.get("kv_heads", H)
        rows, at = p.w_in @ xp, 0
        order = list(range(dk))
        if l["type"] == "retention":          # rotary pairs side by side
            half = mix["rot"]["dims"] // 2
            order = [c for a in range(half) for c in (a, a + half)] + list(range(2 * half, dk))
        for name_, n, dim in (("q", H, dk), ("k", G, dk), ("v", G, dv)) + ((("g", H, dv),) if l["type"] == "retention" else ()):
            got, want = heads(rows[at: at + n * up8(dim)], n, dim), w[pre + "mix." + name_] @ x
            if name_ in "qk":
                want = want.view(n, dim)[:, order].reshape(-1)
            assert torch.allclose(got, want, atol=1e-4), name_
            at += n * up8(dim)
        assert at == rows.numel()
        o, op = rand(H, dv, seed=4).float(), torch.zeros(H, up8(dv))
        op[:, :dv] = o
        y = p.w_o @ op.view(-1)
        assert torch.allclose(y[:W], w[pre + "mix.o"] @ o.view(-1), atol=1e-4) and not y[W:].any()
        n = mod.packed()
        assert n.norm1 is ops.PLAIN and n.norm2 is ops.PLAIN
        assert torch.allclose(n.norm1b[:W], cfg["residual_mult"] * w[pre + "norm1"]) and not n.norm1b[W:].any()
        if l["type"] == "attention":
            c = mod.mixer.constants().prep
            assert (c.n_q, c.n_k, c.eps) == (H * dk, G * dk, cfg["norm"]["eps"])
            assert torch.equal(heads(c.q_norm, H, dk), w[pre + "mix.q.norm"]) and torch.equal(heads(c.k_norm, G, dk), w[pre + "mix.k.norm"])
        if l["mlp"] is not None:
            q, ff = mod.mlp.packed(), l["mlp"]["expert"]["ff"]
            e = l["mlp"]["router"]["experts"] - 1
            up = q.w_gu[e] @ xp
            assert torch.allclose(up[:ff], w[f"{pre}mlp.e{e}.up"] @ x, atol=1e-4) and not up[ff:].any()
    assert torch.allclose(m.packed().final_norm[:W], cfg["logit_scale"] * w["final.norm"])


@pytest.mark.parametrize("rot", [{"base": 500.0, "dims": 6}, {"base": 500.0, "dims": 16, "scaling": P.yarn(4.0, 500, 9.0, 1.5)},
                                 {"base": 30.0, "dims": 4, "scaling": P.yarn(2.0, 10, 1.0, 1.0)}])
def test_rotary_table(rot):
    from vyomai_amd.layers.positional_embeddings import PairRotary
    r = PairRotary(rot["base"], rot["dims"], rot.get("scaling"))
    t = r.table(300, "cpu")
    f, c = O.frequencies(rot)
    want = torch.arange(300, dtype=torch.float64)[:, None] * torch.tensor(f, dtype=torch.float64)
    assert torch.equal(t[:300], torch.stack((c * want.cos(), c * want.sin()), -1).float())
    plain = PairRotary(rot["base"], rot["dims"]).table(300, "cpu")
    assert (plain is t) == ("scaling" not in rot)          # layers of equal constants share a table, others do not


def test_ring_bookkeeping_with_kept_tokens():
    from vyomai_amd import SlotCache
    c = SlotCache([("window", (2, 8, 9, 3)), ("window", (1, 8, 100, 20))], torch.float32, "cpu", slots=1, capacity=2)
    assert c.buffers[0].shape == (1, 2, 4, 8) and c.buffers[1].shape == (1, 1, 21, 8)    # never fewer rows than kept tokens + 1
    [a] = c.allocate(1)
    c.reserve([a], [4])
    c.advance([a], [4])
    for b in c.buffers:
        b[a, :, :4] = torch.arange(4.0)[None, :, None]
    c.reserve([a], [30])
    assert c.buffers[0].shape[2] == 9 and c.buffers[1].shape[2] == c.capacity == 34
    for b in c.buffers:
        assert torch.equal(b[a, 0, :4, 0], torch.arange(4.0)) and not b[a, :, 4:].any()
    c.reserve([a], [500])
    assert [b.shape[2] for b in c.buffers] == [9, 100]


def test_argument_errors_without_a_gpu():
    from vyomai_amd import _lib
    buf = (ctypes.c_char * 4096)()
    p = (ctypes.addressof(buf) + 63) // 64 * 64
    prep = _lib.VyQkvPrep(p, p, 8, 8, 1e-5, 0.0)

    def rows(ring=p, R=4, keep=1, dims=0, length=0, prep=prep, ldp=64):
        _lib.call("vy_qkv_rows", p, ldp, 0, 8, 16, ctypes.byref(prep) if prep else None, ring, 64, 64, R, keep, p, dims, length, 1, None, p,
                  None, 1, 1, 1, 1, 8, 8, 1, None)
    for kw, match in (({"keep": 4}, "4 kept of 4 rows"), ({"dims": 10, "length": 5}, "rotary table"), ({"prep": None}, "bad arguments"),
                      ({"ldp": 60}, "bad arguments"), ({"R": 5}, "ring strides"),
                      ({"prep": _lib.VyQkvPrep(p, None, 8, 8, 1e-5, 0.0)}, "norms"),
                      ({"prep": _lib.VyQkvPrep(p, p, 9, 8, 1e-5, 0.0)}, "norms"),
                      ({"prep": _lib.VyQkvPrep(None, None, 0, 0, 0.0, 0.5, p, 8, 7, 6, 8)}, "value rows")):
        with pytest.raises(_lib.VyomHipError, match=match):
            rows(**kw)
    with pytest.raises(_lib.VyomHipError, match="rotary table"):
        _lib.call("vy_decay_attn", p, 24, 0, 8, 16, p, p, None, p, None, p, 8, 1, 1, 1, 8, 8, 1, p, 10, 4, 1.0, None, 0, 1, None)
    with pytest.raises(_lib.VyomHipError, match="multiples of 8"):
        _lib.call("vy_head_norm_gate", p, 8, None, p, 8, p, 8, 1, 1, 5, 6, 1e-5, 1, None)
    moe = _lib.VyMoe(4, 2, 2, 1, 8, 8, 2, 0, 1, 1, 1.0, 1.0, 1.0, p, p, p)
    for field, value in (("act", 2), ("score", 2), ("group_best", 3)):
        moe.act, moe.score, moe.group_best = 0, 0, 1
        setattr(moe, field, value)
        with pytest.raises(_lib.VyomHipError, match="activation"):
            _lib.call("vy_moe_fwd", ctypes.byref(moe), p, 8, 1, None, 1, p, 8, p, p, p, p, 4096, 1, None)
    win = _lib.VyAttnWindow(4, 0, 0, 8, None, 0, 0, -1)
    with pytest.raises(_lib.VyomHipError, match="-1 kept keys"):
        _lib.call("vy_attn_fwd_ex", p, 8, 8, 8, p, 8, 8, 8, p, 8, 8, 8, p, 8, 8, None, 0, 0, None, None, 1, 1, 1, 1, 1, 8, 8, 1.0,
                  ctypes.byref(win), 1, None)
