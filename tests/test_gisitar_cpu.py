"""Gisitar without a GPU: the oracle against closed forms, checkpoint reading and naming, packing, slot bookkeeping, and
that the product path refuses to run on the CPU."""
import json
import os
import struct
import subprocess
import sys

import pytest
import torch

from oracle import gisitar_oracle as O
from tests import gisitar_cases as G

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


def test_oracle_recurrence_equals_the_weighted_sum():
    g = torch.Generator().manual_seed(0)
    T, dk, dv, d = 9, 4, 5, 0.6
    q, k, v = (torch.randn(T, n, generator=g, dtype=torch.float64) for n in (dk, dk, dv))
    o, s = O.decayed_recurrence(q, k, v, d)
    for t in range(T):
        direct = sum(d ** (t - j) * (q[t] @ k[j]) * v[j] for j in range(t + 1))
        assert torch.allclose(o[t], direct, atol=1e-12)
    o2, s2 = O.decayed_recurrence(q[4:], k[4:], v[4:], d, O.decayed_recurrence(q[:4], k[:4], v[:4], d)[1])
    assert torch.allclose(o[4:], o2) and torch.allclose(s, s2)


def test_oracle_attention_is_the_masked_softmax():
    g = torch.Generator().manual_seed(1)
    q, k, v = (torch.randn(6, n, generator=g, dtype=torch.float64) for n in (3, 3, 4))
    s = (q @ k.T) * 0.7
    s = s.masked_fill(torch.ones(6, 6).triu(1).bool(), float("-inf"))
    assert torch.allclose(O.softmax_attention(q, k, v, 0.7), s.softmax(-1) @ v)


@pytest.mark.parametrize("name", list(G.CONFIGS))
def test_oracle_is_causal(name):
    cfg, w = G.CONFIGS[name], G.weights(G.CONFIGS[name])
    ids = G.tokens(cfg, 12)
    full = O.forward(w, cfg, ids)
    assert torch.allclose(full[:7], O.forward(w, cfg, ids[:7]), atol=1e-12)
    other = list(ids)
    other[2] = (other[2] + 1) % cfg["vocab"]
    assert not torch.allclose(full[11], O.forward(w, cfg, other)[11], atol=1e-6)


@pytest.mark.parametrize("name", list(G.CONFIGS))
def test_checkpoint_loads_by_name(name, tmp_path):
    from vyomai_amd import GisitarModel, load_pretrained
    cfg, w = G.CONFIGS[name], G.weights(G.CONFIGS[name])
    G.write_folder(tmp_path, cfg, w)
    m = load_pretrained(str(tmp_path), torch.float32, "cpu")
    assert isinstance(m, GisitarModel)
    named = {m.checkpoint_name(n): p for n, p in m.named_parameters()}
    assert set(named) == set(w)
    for n, t in w.items():
        assert torch.equal(named[n], t), n


def test_checkpoint_errors(tmp_path):
    from vyomai_amd import load_pretrained
    cfg, w = G.CONFIGS["edges"], G.weights(G.CONFIGS["edges"])
    G.write_folder(tmp_path, cfg, {n: t for n, t in w.items() if n != "l1.mix.norm"})
    with pytest.raises(KeyError, match="l1.mix.norm"):
        load_pretrained(str(tmp_path), torch.float32, "cpu")
    G.write_folder(tmp_path, cfg, {**w, "l9.extra": torch.zeros(2)})
    with pytest.raises(KeyError, match="l9.extra"):
        load_pretrained(str(tmp_path), torch.float32, "cpu")
    G.write_folder(tmp_path, cfg, {**w, "head": w["head"][:-1]})
    with pytest.raises(ValueError, match="head"):
        load_pretrained(str(tmp_path), torch.float32, "cpu")
    G.write_folder(tmp_path, {**cfg, "architecture": "Nobody"}, w)
    with pytest.raises(ValueError, match="Nobody"):
        load_pretrained(str(tmp_path), torch.float32, "cpu")
    G.write_folder(tmp_path, {**cfg, "layers": [{**cfg["layers"][0], "type": "sieve"}]}, w)
    with pytest.raises(ValueError, match="sieve"):
        load_pretrained(str(tmp_path), torch.float32, "cpu")


def test_safetensors_reader(tmp_path):
    from vyomai_amd.models.registry import read_safetensors
    a, b = torch.arange(6, dtype=torch.float32).view(2, 3), torch.tensor([7, -1], dtype=torch.int32)
    head = json.dumps({"__metadata__": {"x": "y"}, "a": {"dtype": "F32", "shape": [2, 3], "data_offsets": [0, 24]},
                       "b": {"dtype": "I32", "shape": [2], "data_offsets": [24, 32]}}).encode()
    f = tmp_path / "t.safetensors"
    f.write_bytes(struct.pack("<Q", len(head)) + head + a.numpy().tobytes() + b.numpy().tobytes())
    got = read_safetensors(str(f))
    assert set(got) == {"a", "b"} and torch.equal(got["a"], a) and torch.equal(got["b"], b)
    f.write_bytes(struct.pack("<Q", len(head)) + head + a.numpy().tobytes())
    with pytest.raises(ValueError, match="'b'"):
        read_safetensors(str(f))


@pytest.mark.parametrize("name", list(G.CONFIGS))
def test_packed_weights_are_the_weights_with_zero_padding(name, tmp_path):
    from vyomai_amd import load_pretrained
    from vyomai_amd.ops import up8
    cfg, w = G.CONFIGS[name], G.weights(G.CONFIGS[name])
    G.write_folder(tmp_path, cfg, w)
    m = load_pretrained(str(tmp_path), torch.float32, "cpu")
    W = cfg["width"]
    x = torch.randn(W, generator=torch.Generator().manual_seed(3))
    xp = torch.zeros(up8(W))
    xp[:W] = x
    for i, l in enumerate(cfg["layers"]):
        mix, p = l["mixer"], m.layers[i].mixer.packed()
        H, dv = mix["heads"], mix["vdim"]
        rows = p.w_in @ xp
        gate = rows[-H * up8(dv):].view(H, up8(dv))
        assert torch.allclose(gate[:, :dv].reshape(-1), w[f"l{i}.mix.g"] @ x, atol=1e-4) and not gate[:, dv:].any()
        y = torch.zeros(H, up8(dv))
        y[:, :dv] = torch.randn(H, dv)
        out = p.w_o @ y.view(-1)
        assert torch.allclose(out[:W], w[f"l{i}.mix.o"] @ y[:, :dv].reshape(-1), atol=1e-4) and not out[W:].any()
        for t in vars(p).values():
            assert not isinstance(t, torch.Tensor) or t.dim() != 2 or t.shape[-1] % 8 == 0 or t is p.__dict__.get("decay_pow")
    # a changed parameter is packed anew
    mixer = m.layers[0].mixer
    before = mixer.packed().w_o.clone()
    with torch.no_grad():
        mixer.out.weight.mul_(2)
    assert torch.equal(mixer.packed().w_o, 2 * before)


def test_decay_powers_are_rounded_once():
    from vyomai_amd.layers.lightning_attention import LightningAttention
    m = LightningAttention(8, 3, 8, 8, (0.999, 0.0, 1.0), 1e-5)
    t = m.packed().decay_pow
    assert t.dtype == torch.float32
    assert t[0, 64].item() == torch.tensor(0.999 ** 64, dtype=torch.float64).float().item()
    assert t[1, 0] == 1 and not t[1, 1:].any() and bool((t[2] == 1).all())
    with pytest.raises(ValueError, match="2 decays for 3 heads"):
        LightningAttention(8, 3, 8, 8, (0.5, 0.5), 1e-5)


def test_slot_cache_bookkeeping():
    from vyomai_amd import SlotCache
    c = SlotCache([("latent", 8), ("state", (2, 3, 4))], torch.float32, "cpu", slots=2, capacity=4)
    a, b = c.allocate(2)
    assert {a, b} == {0, 1} and c.free_slots == 0
    batch = c.reserve([a, b], [3, 1])
    assert batch.fresh and batch.max_keys == 3 and batch.count.tolist() == [3, 1]
    c.advance([a, b], [3, 1])
    assert c.lengths.tolist() == c.length and c.length[a] == 3
    c.buffers[0][a, :3] = 5.0
    c.buffers[1][a] = 6.0
    gen = c.generation
    batch = c.reserve([a], [2])                       # 5 > 4 rows: grows, keeps what is there
    assert c.capacity >= 5 and c.generation == gen + 1 and not batch.fresh and batch.max_keys == 5 and batch.count is None
    assert bool((c.buffers[0][a, :3] == 5).all()) and not c.buffers[0][a, 3:].any()
    [d] = c.allocate(1)                               # more slots
    assert d not in (a, b) and c.slots >= 3 and bool((c.buffers[1][a] == 6).all()) and c.lengths[a] == 3
    c.free([a])
    with pytest.raises(ValueError, match="not in use"):
        c.free([a])
    again = c.allocate(1)[0]
    assert again == a and c.length[a] == 0 and c.lengths[a] == 0     # handed on empty, the old rows need no clearing
    with pytest.raises(ValueError, match="once"):
        c.reserve([a, a], [1, 1])
    with pytest.raises(ValueError, match="at least one"):
        c.reserve([a, b], [0, 1])


def test_padding_must_follow_the_tokens():
    from vyomai_amd.models.hybrid import HybridDecoderModel as M
    ids = torch.zeros(2, 4, dtype=torch.long)
    assert M._counts(ids, torch.tensor([[1, 1, 0, 0], [1, 1, 1, 1]])) == [2, 4]
    for bad in ([[0, 1, 1, 1], [1, 1, 1, 1]], [[0, 0, 0, 0], [1, 1, 1, 1]]):
        with pytest.raises(ValueError, match="padding"):
            M._counts(ids, torch.tensor(bad))


def test_no_cpu_path(tmp_path):
    from vyomai_amd import load_pretrained
    from vyomai_amd._lib import VyomHipError
    cfg = G.CONFIGS["edges"]
    G.write_folder(tmp_path, cfg, G.weights(cfg))
    m = load_pretrained(str(tmp_path), torch.float32, "cpu")
    with pytest.raises(VyomHipError, match="CPU"):
        m(torch.zeros(1, 4, dtype=torch.long))


def test_argument_errors_without_a_gpu():
    import ctypes
    from vyomai_amd import _lib
    buf = (ctypes.c_char * 4096)()
    p = (ctypes.addressof(buf) + 63) // 64 * 64
    with pytest.raises(_lib.VyomHipError, match="multiples of 4"):
        _lib.call("vy_residual_norm", p, 8, p, 8, None, 0, None, 0, None, None, 1e-5, p, 1e-5, p, 8, 1, 5, 6, 0, 1, None)
    with pytest.raises(_lib.VyomHipError, match="multiples of 8"):
        _lib.call("vy_latent_decode", p, 8, p, p, p, 8, 8, None, p, 1, p, 8, None, 0, 0, 0, 1, 1, 8, 8, 12, 1.0, p, 4096, 1, None)
    with pytest.raises(_lib.VyomHipError, match="workspace"):
        _lib.call("vy_latent_decode", p, 8, p, p, p, 8, 8, None, p, 1, p, 8, None, 0, 0, 0, 1, 1, 8, 8, 8, 1.0, p, 16, 1, None)
    with pytest.raises(_lib.VyomHipError, match="multiples of 8"):
        _lib.call("vy_decay_attn", p, 24, 0, 8, 20, p, p, None, p, None, p, 8, 1, 1, 1, 8, 8, 1, None, 0, 0, 1.0, None, 0, 1, None)
    with pytest.raises(_lib.VyomHipError, match="null"):
        _lib.call("vy_hybrid_decoder_step", None, p, None, p, 1, p, 8, None)


def test_trace_command_line():
    r = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--help"], capture_output=True, text=True)
    assert r.returncode == 0 and "--max-tokens" in r.stdout
    assert os.access(os.path.join(ROOT, "bin", "trace_run"), os.X_OK)
