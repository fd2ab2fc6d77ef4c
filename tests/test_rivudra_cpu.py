"""Rivudra without a GPU: the oracle against closed forms, checkpoint loading with stacked experts, packing, the ring's
bookkeeping, and argument checks of the C ABI."""
import ctypes

import pytest
import torch

from oracle import rivudra_oracle as O
from tests import rivudra_cases as R


def test_oracle_window_attention_is_the_banded_softmax_with_a_sink():
    g = torch.Generator().manual_seed(1)
    T, W = 9, 4
    q, k, v = (torch.randn(T, n, generator=g, dtype=torch.float64) for n in (3, 3, 5))
    s = (q @ k.T) * 0.7
    i, j = torch.arange(T)[:, None], torch.arange(T)[None]
    s = s.masked_fill((j > i) | (i - j >= W), float("-inf"))
    s = torch.cat([s, torch.zeros(T, 1, dtype=torch.float64)], 1)           # the sink: score 0, value 0
    want = s.softmax(-1) @ torch.cat([v, torch.zeros(1, 5, dtype=torch.float64)])
    assert torch.allclose(O.window_attention(q, k, v, 0.7, W), want)


def test_oracle_rotation_keeps_lengths_and_depends_on_distance():
    g = torch.Generator().manual_seed(2)
    q, k = (torch.randn(1, 10, generator=g, dtype=torch.float64) for _ in range(2))
    a = O.rotate(q, 50.0, 6, 11)
    assert torch.allclose(a.norm(), q.norm()) and torch.equal(a[:, 6:], q[:, 6:]) and not torch.allclose(a[:, :6], q[:, :6])
    assert torch.allclose(O.rotate(q, 50.0, 6, 0), q)
    dot = [(O.rotate(q, 50.0, 6, p + 3) * O.rotate(k, 50.0, 6, p)).sum() for p in (0, 5, 40)]
    assert torch.allclose(dot[0], dot[1]) and torch.allclose(dot[0], dot[2])


def test_oracle_routing():
    cfg = {"experts": 6, "top": 2, "scale": 2.0, "groups": {"count": 3, "keep": 1}}
    z = torch.tensor([0.0, 3.0, 2.9, 2.8, 1.0, 2.0], dtype=torch.float64)     # groups (0, 1), (2, 3), (4, 5)
    chosen, w = O.route(z, cfg)
    assert chosen == [1, 0] and abs(sum(w) - 2.0) < 1e-12
    assert abs(w[0] / w[1] - torch.exp(torch.tensor(3.0)).item()) < 1e-4
    cfg["groups"]["keep"] = 2
    assert O.route(z, cfg)[0] == [1, 2]


@pytest.mark.parametrize("name", list(R.CONFIGS))
def test_oracle_is_causal(name):
    cfg, w = R.CONFIGS[name], R.weights(R.CONFIGS[name])
    ids = R.tokens(cfg, 8)
    full = O.forward(w, cfg, ids)
    assert torch.allclose(full[:5], O.forward(w, cfg, ids[:5]), atol=1e-12)


@pytest.mark.parametrize("name", list(R.CONFIGS))
def test_checkpoint_loads_by_name_and_stacks_the_experts(name, tmp_path):
    from vyomai_amd import RivudraModel, load_pretrained
    cfg, w = R.CONFIGS[name], R.weights(R.CONFIGS[name])
    R.write_folder(tmp_path, cfg, w)
    m = load_pretrained(str(tmp_path), torch.float32, "cpu")
    assert isinstance(m, RivudraModel)

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
            assert l.mlp.gate.untyped_storage().data_ptr() == p.w_gu.untyped_storage().data_ptr() == l.mlp.up.untyped_storage().data_ptr()
            assert l.mlp.packed() is p
    check()


def test_checkpoint_errors(tmp_path):
    from vyomai_amd import load_pretrained
    cfg, w = R.CONFIGS["edges"], R.weights(R.CONFIGS["edges"])
    R.write_folder(tmp_path, cfg, {n: t for n, t in w.items() if n != "l1.mlp.e2.up"})
    with pytest.raises(KeyError, match="l1.mlp.e2.up"):
        load_pretrained(str(tmp_path), torch.float32, "cpu")
    R.write_folder(tmp_path, cfg, {**w, "l1.mlp.e2.up": w["l1.mlp.e2.up"][:-1]})
    with pytest.raises(ValueError, match="l1.mlp.e2.up"):
        load_pretrained(str(tmp_path), torch.float32, "cpu")
    R.write_folder(tmp_path, cfg, {**w, "l1.mlp.e4.up": w["l1.mlp.e2.up"]})      # one expert too many
    with pytest.raises(KeyError, match="l1.mlp.e4.up"):
        load_pretrained(str(tmp_path), torch.float32, "cpu")
    bad = dict(cfg["layers"][1], mlp=dict(cfg["layers"][1]["mlp"], kind="sieve"))
    R.write_folder(tmp_path, {**cfg, "layers": [bad]}, w)
    with pytest.raises(ValueError, match="sieve"):
        load_pretrained(str(tmp_path), torch.float32, "cpu")


def test_impossible_sizes_are_refused():
    from vyomai_amd.layers.ffn import MixtureFeedForward
    from vyomai_amd.layers.window_attention import WindowAttention
    for kw in ({"top": 5}, {"groups": 3}, {"groups": 2, "keep": 3}, {"top": 3, "groups": 2, "keep": 1}):
        with pytest.raises(ValueError, match="experts"):
            MixtureFeedForward(8, 4, **{"top": 1, "inner": 8, "limit": 1.0, **kw})
    with pytest.raises(ValueError, match="heads"):
        WindowAttention(8, 3, 2, 8, 8, 1.0, 4)
    for kw in ({"window": 0}, {"scale": -1.0}, {"rot_dims": 10}, {"rot_dims": 3}):
        with pytest.raises(ValueError):
            WindowAttention(8, 2, 1, 8, 8, **{"scale": 1.0, "window": 4, **kw})


@pytest.mark.parametrize("name", list(R.CONFIGS))
def test_fused_products_are_the_separate_ones(name, tmp_path):
    from vyomai_amd import load_pretrained
    from vyomai_amd.ops import up8
    cfg, w = R.CONFIGS[name], R.weights(R.CONFIGS[name])
    R.write_folder(tmp_path, cfg, w)
    m = load_pretrained(str(tmp_path), torch.float32, "cpu")
    W = cfg["width"]
    g = torch.Generator().manual_seed(3)
    x = torch.randn(W, generator=g)
    xp = torch.zeros(up8(W))
    xp[:W] = x

    def heads(rows, n, dim):
        r = rows.view(n, up8(dim))
        assert not r[:, dim:].any()
        return r[:, :dim].reshape(-1)

    for i, l in enumerate(cfg["layers"]):
        mix, p, pre = l["mixer"], m.layers[i].packed(), f"l{i}."
        H, G, dk, dv = mix["heads"], mix["kv_heads"], mix["dim"], mix["vdim"]
        rows, at = p.w_in @ xp, 0
        for name_, n, dim in (("q", H, dk), ("k", G, dk), ("v", G, dv), ("g", H, dv)):
            part = rows[at: at + n * up8(dim)]
            assert torch.allclose(heads(part, n, dim), w[pre + "mix." + name_] @ x, atol=1e-4)
            at += n * up8(dim)
        assert at == p.n_mix
        o = torch.randn(H, dv, generator=g)
        both, want = torch.zeros(H, up8(dv)), w[pre + "mix.o"] @ o.view(-1)
        both[:, :dv] = o
        both = both.view(-1)
        if l["mlp"] is not None and "shared" in l["mlp"]:
            ff = l["mlp"]["shared"]["ff"]
            gu = rows[at:].view(2, up8(ff))
            assert torch.allclose(gu[0, :ff], w[pre + "mlp.shared.gate"] @ x, atol=1e-4)
            assert torch.allclose(gu[1, :ff], w[pre + "mlp.shared.up"] @ x, atol=1e-4) and not gu[:, ff:].any()
            a = torch.randn(ff, generator=g)
            both = torch.cat([both, a, torch.zeros(up8(ff) - ff)])
            want = want + w[pre + "mlp.shared.down"] @ a
        else:
            assert at == rows.numel()
        y = p.w_o @ both
        assert torch.allclose(y[:W], want, atol=1e-4) and not y[W:].any()
        assert torch.allclose(p.norm1[:W], 1 + w[pre + "norm1"]) and not p.norm1[W:].any()
        if l["mlp"] is not None:
            q, ff = m.layers[i].mlp.packed(), l["mlp"]["expert"]["ff"]
            e = l["mlp"]["router"]["experts"] - 1
            gu = (q.w_gu[e] @ xp).view(-1, 2)
            assert torch.allclose(gu[:ff, 0], w[f"{pre}mlp.e{e}.gate"] @ x, atol=1e-4) and not gu[ff:].any()
            assert torch.allclose(gu[:ff, 1], w[f"{pre}mlp.e{e}.up"] @ x, atol=1e-4)


def test_rotary_table():
    from vyomai_amd.layers.positional_embeddings import PairRotary
    r = PairRotary(500.0, 6)
    t = r.table(3, "cpu")
    assert t.dtype == torch.float32 and t.shape[1:] == (3, 2) and t.shape[0] >= 3
    a = torch.tensor(2 * 500.0 ** (-4 / 6), dtype=torch.float64)
    assert t[2, 2, 0].item() == a.cos().float().item() and t[2, 2, 1].item() == a.sin().float().item()
    big = r.table(5000, "cpu")
    assert big.shape[0] >= 5000 and torch.equal(big[: t.shape[0]], t) and r.table(10, "cpu") is big
    assert PairRotary(500.0, 0).table(10, "cpu") is None
    with pytest.raises(ValueError):
        PairRotary(500.0, 5)


def test_ring_bookkeeping():
    from vyomai_amd import SlotCache
    c = SlotCache([("window", (2, 8, 6)), ("window", (1, 8, 100))], torch.float32, "cpu", slots=1, capacity=4)
    assert c.buffers[0].shape == (1, 2, 4, 8) and c.buffers[1].shape == (1, 1, 4, 8)
    [a] = c.allocate(1)
    assert c.reserve([a], [4]).past == 0
    c.advance([a], [4])
    for b in c.buffers:
        b[a, :, :4] = torch.arange(4.0)[None, :, None]
    batch = c.reserve([a], [1])                      # grows: the short ring to its window, the long one with the capacity
    assert batch.past == 4 and not batch.fresh and c.buffers[0].shape[2] == 6 and c.buffers[1].shape[2] == c.capacity == 8
    for b in c.buffers:
        assert torch.equal(b[a, 0, :4, 0], torch.arange(4.0)) and not b[a, :, 4:].any()
    c.advance([a], [1])
    same = c.buffers[0]
    c.reserve([a], [50])
    assert c.buffers[0] is same and c.buffers[1].shape[2] == c.capacity      # a full window never grows again
    c.allocate(1)
    assert c.buffers[0].shape[:3] == (2, 2, 6) and torch.equal(c.buffers[0][a, 0, :4, 0], torch.arange(4.0))


def test_argument_errors_without_a_gpu():
    from vyomai_amd import _lib
    buf = (ctypes.c_char * 4096)()
    p = (ctypes.addressof(buf) + 63) // 64 * 64
    win = [p, 64, 0, 8, 16, 24, p, 64, 64, 4, 0, None, 0, 0, None, None, None, p, 1, p, 8, 1, 1, 1, 8, 8]

    def decode(**kw):
        a = list(win)
        for i, v in kw.items():
            a[int(i[1:])] = v
        return a
    with pytest.raises(_lib.VyomHipError, match="ring strides"):
        _lib.call("vy_window_decode", *decode(_8=56, _7=56), 1.0, 1, None, 0, 1, None)
    with pytest.raises(_lib.VyomHipError, match="rotary table"):
        _lib.call("vy_window_decode", *decode(_11=p, _12=10, _13=5), 1.0, 1, None, 0, 1, None)
    with pytest.raises(_lib.VyomHipError, match="5 positions, rotary table of 4"):
        _lib.call("vy_window_decode", *decode(_11=p, _12=8, _13=4, _18=5), 1.0, 1, None, 0, 1, None)
    with pytest.raises(_lib.VyomHipError, match="bad arguments"):
        _lib.call("vy_window_decode", *win, 0.0, 1, None, 0, 1, None)
    with pytest.raises(_lib.VyomHipError, match="4 kept of 4 rows"):
        _lib.call("vy_window_decode", *decode(_10=4), 1.0, 1, None, 0, 1, None)
    with pytest.raises(_lib.VyomHipError, match="multiples of 8"):
        _lib.call("vy_window_decode", *decode(_2=4), 1.0, 1, None, 0, 1, None)
    moe = _lib.VyMoe(4, 3, 2, 1, 8, 8, 0, 0, 1, 1, 1.0, 1.0, 1.0, p, p, p)
    with pytest.raises(_lib.VyomHipError, match="3 of 4 experts, 1 of 2 groups"):
        _lib.call("vy_moe_fwd", ctypes.byref(moe), p, 8, 1, None, 1, p, 8, p, p, p, p, 4096, 1, None)
    moe.top = 2
    with pytest.raises(_lib.VyomHipError, match="workspace"):
        _lib.call("vy_moe_fwd", ctypes.byref(moe), p, 8, 1, None, 1, p, 8, p, p, p, p, 16, 1, None)
    with pytest.raises(_lib.VyomHipError, match="routed rows"):
        rows = _lib.VyRoutedRows(p, 8, p, None, 2)
        _lib.call("vy_residual_norm_routed", p, 8, p, 8, None, 0, None, 0, None, 1.0, ctypes.byref(rows), None, 1e-5, p, 1e-5, p, 8,
                  1, 8, 8, 1, 1, None)


def test_layout_of_the_plan_structures():
    """ctypes mirrors against the sizes a C compiler gives the header's structs."""
    import os
    import subprocess
    import tempfile
    from vyomai_amd import _lib, decode_plan as D
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    names = {"vy_hybrid_layer": D.VyHybridLayer, "vy_hybrid_plan": D.VyHybridPlan, "vy_moe": _lib.VyMoe,
             "vy_attn_window": _lib.VyAttnWindow, "vy_qkv_prep": _lib.VyQkvPrep, "vy_routed_rows": _lib.VyRoutedRows}
    src = "#include <stdio.h>\n#include <stddef.h>\n#include \"vyom_hip.h\"\nint main(){\n"
    for n, cls in names.items():
        fields = [f[0].rstrip("_") for f in cls._fields_]    # (lambda_: a keyword in Python)
        src += f'printf("%zu", sizeof({n}));\n' + "".join(f'printf(" %zu", offsetof({n}, {f}));\n' for f in fields)
        src += 'printf("\\n");\n'
    with tempfile.TemporaryDirectory() as d:
        with open(os.path.join(d, "t.c"), "w") as f:
            f.write(src + "return 0;}\n")
        subprocess.run(["gcc", "-I", os.path.join(root, "include"), os.path.join(d, "t.c"), "-o", os.path.join(d, "t")], check=True)
        lines = subprocess.run([os.path.join(d, "t")], check=True, capture_output=True, text=True).stdout.splitlines()
    for (n, cls), line in zip(names.items(), lines):
        assert [int(v) for v in line.split()] == [ctypes.sizeof(cls)] + [getattr(cls, f[0]).offset for f in cls._fields_], n
