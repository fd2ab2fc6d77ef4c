"""Gisitar on the GPU: every mechanism alone and the whole model (prefill, decode, portions, unequal batches, slots used
again, generation, trace replay) against the plain oracle."""
import json
import os
import subprocess
import sys

import pytest
import torch

from oracle import gisitar_oracle as O
from tests import gisitar_cases as G

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
DT = [torch.float32, torch.bfloat16]
TOL = {torch.float32: 2e-5, torch.bfloat16: 1.2e-2}


def rnd(*shape, seed=0, scale=1.0):
    """fp64 values representable in bf16."""
    g = torch.Generator().manual_seed(seed)
    return (torch.randn(*shape, generator=g) * scale).to(torch.bfloat16).double()


def close(got, want, dt, tol=None):
    got = got.double().cpu()
    err = (got - want).abs().max().item() / max(want.abs().max().item(), 1e-30)
    assert torch.isfinite(got).all() and err < (tol or TOL[dt]), err


def pad_cols(t, n):
    out = torch.zeros(*t.shape[:-1], n, dtype=t.dtype)
    out[..., : t.shape[-1]] = t
    return out


def up8(n):
    return (n + 7) // 8 * 8


# ---- norms ----------------------------------------------------------------------------------------
@pytest.mark.parametrize("dt", DT)
@pytest.mark.parametrize("rms", [False, True])
@pytest.mark.parametrize("M,N", [(3, 37), (1, 1), (5, 256), (1100, 53), (1030, 1500), (2, 5000)])
def test_residual_norm(dt, rms, M, N):
    from vyomai_amd import ops
    NP, eps = up8(N), 1e-3
    x, y = rnd(M, N, seed=1) + 3.0, (rnd(M, N, seed=2) + 0.5).to(torch.bfloat16).double()
    a, b = 1 + 0.3 * rnd(N, seed=3), 1 + 0.3 * rnd(N, seed=4)
    norm = O.rms_norm if rms else O.layer_norm
    wx = x + norm(y, a, eps)
    xd = pad_cols(x, NP).float().cuda()
    h = ops.residual_norm(xd, N, y=pad_cols(y, NP).to(dt).cuda(), post=pad_cols(a, NP).float().cuda(),
                          pre=pad_cols(b, NP).float().cuda(), eps=eps, rms=rms)
    close(xd[:, :N], wx, torch.float32)
    if N > 1:
        close(h[:, :N], norm(wx, b, eps), dt)
    assert not xd[:, N:].any() and not h[:, N:].any()
    # plain add, norm only, embedding
    x1 = pad_cols(x, NP).float().cuda()
    assert ops.residual_norm(x1, N, y=pad_cols(y, NP).to(dt).cuda(), eps=eps) is None
    close(x1[:, :N], x + y, torch.float32)
    table = pad_cols(rnd(9, N, seed=5), NP)
    ids = torch.arange(M) % 11                     # 9 and 10 are outside the vocabulary
    flag = torch.zeros(1, dtype=torch.int32, device="cuda")
    x2 = torch.full((M, NP), 7.0, device="cuda")
    h = ops.residual_norm(x2, N, table=table.to(dt).cuda(), ids=ids.cuda(), pre=pad_cols(b, NP).float().cuda(), eps=eps,
                          rms=rms, err_flag=flag)
    want = torch.where((ids < 9)[:, None], table[ids.clamp(max=8)][:, :N], torch.zeros(1, dtype=torch.float64))
    close(x2[:, :N], want, torch.float32)
    assert int(flag) == int(M > 9)
    if N > 1:
        close(h[:, :N], norm(want, b, eps), dt)


def test_layer_norm_of_a_large_mean_keeps_its_variance():
    """Deviations are squared about the mean: a mean of 300 over a spread of 0.01 is nothing special."""
    from vyomai_amd import ops
    x = 300.0 + 0.01 * rnd(4, 64, seed=1)
    w = torch.ones(64, dtype=torch.float64)
    xd = x.float().cuda()
    h = ops.residual_norm(xd, 64, pre=w.float().cuda(), eps=1e-6, dtype=torch.float32)
    close(h, O.layer_norm(xd.double().cpu(), w, 1e-6), torch.float32, 1e-3)


@pytest.mark.parametrize("dt", DT)
@pytest.mark.parametrize("nq,nc", [(21, 27), (8, 8), (600, 100), (64, 2100)])
def test_latent_norm_and_its_cache_rows(dt, nq, nc):
    from vyomai_amd import ops
    B, L, npq, npc, eps = 3, 4, up8(nq), up8(nc), 1e-5
    p = torch.cat([pad_cols(rnd(B * L, nq, seed=1), npq), pad_cols(rnd(B * L, nc, seed=2), npc), rnd(B * L, 8)], -1)
    wq, wc = 1 + 0.3 * rnd(nq, seed=3), 1 + 0.3 * rnd(nc, seed=4)
    cache = torch.full((5, 9, npc), -7.0, dtype=dt, device="cuda")
    start = torch.tensor([2, 0, 5, 0, 7], dtype=torch.int32, device="cuda")
    slots = torch.tensor([4, 1, 2], dtype=torch.int32, device="cuda")
    count = torch.tensor([2, 4, 3], dtype=torch.int32, device="cuda")     # slot 4: rows 7, 8 of 9
    q, c = ops.latent_norm(p.to(dt).cuda(), pad_cols(wq, npq).float().cuda(), nq, pad_cols(wc, npc).float().cuda(), nc, B, L,
                           eps, cache=cache, slots=slots, start=start, count=count)
    wantc = O.rms_norm(p[:, npq:npq + nc], wc, eps)
    close(q[:, :nq], O.rms_norm(p[:, :nq], wq, eps), dt)
    close(c[:, :nc], wantc, dt)
    assert not q[:, nq:].any() and not c[:, nc:].any()
    mirror = torch.full((5, 9, npc), -7.0, dtype=dt)
    for b, (s, st, n) in enumerate([(4, 7, 2), (1, 0, 4), (2, 5, 3)]):
        mirror[s, st:st + n] = c.cpu().view(B, L, -1)[b, :n]
    assert torch.equal(cache.cpu(), mirror)


@pytest.mark.parametrize("dt", DT)
@pytest.mark.parametrize("M,N", [(1, 24), (7, 19), (3, 5000)])
def test_rmsnorm_gate(dt, M, N):
    from vyomai_amd import ops
    NP = up8(N)
    x, g, w = rnd(M, N, seed=1), rnd(M, N, seed=2, scale=3.0), 1 + 0.3 * rnd(N, seed=3)
    y = ops.rmsnorm_gate(pad_cols(x, NP).to(dt).cuda(), pad_cols(w, NP).float().cuda(), N, pad_cols(g, NP).to(dt).cuda(), 1e-5)
    close(y[:, :N], O.rms_norm(x, w, 1e-5) * O.sigmoid(g), dt)


# ---- attention ------------------------------------------------------------------------------------
def attention_want(q, k, v, scale, gate, starts):
    """q (B,h,L,dh), k/v (B,h,S,.): row i of sequence b sees keys 0 .. starts[b] + i."""
    B, h, L, _ = q.shape
    out = torch.zeros(B, L, h, v.shape[3], dtype=torch.float64)
    for b in range(B):
        for a in range(h):
            for i in range(L):
                n = starts[b] + i + 1
                s = (k[b, a, :n] @ q[b, a, i]) * scale
                e = torch.exp(s - s.max())
                out[b, i, a] = (e / e.sum()) @ v[b, a, :n]
    out = out.reshape(B, L, -1)
    return out if gate is None else out * O.sigmoid(gate)


@pytest.mark.parametrize("dt", DT)
@pytest.mark.parametrize("dh,dv", [(64, 64), (128, 128), (8, 8), (24, 40), (40, 24), (72, 112), (112, 8), (64, 200), (200, 72),
                                   (256, 256), (16, 136)])
@pytest.mark.parametrize("starts,L", [([0, 0], 70), ([5, 63], 3), ([0, 130], 33)])
def test_attention_with_its_own_value_width(dt, dh, dv, starts, L):
    from vyomai_amd import ops
    B, h, S = 2, 2, max(starts) + L
    q, k, v = rnd(B, h, L, dh, seed=1), rnd(B, h, S, dh, seed=2), rnd(B, h, S, dv, seed=3)
    gate = rnd(B, L, h * dv, seed=4, scale=2.0)
    slots = torch.tensor([3, 1], dtype=torch.int32, device="cuda")
    start = torch.tensor([9, starts[1], 9, starts[0]], dtype=torch.int32, device="cuda")
    scale = dh ** -0.5
    o = ops.attention_ex(q.to(dt).cuda(), k.to(dt).cuda(), v.to(dt).cuda(), scale, gate=gate.to(dt).cuda(), start=start, slots=slots)
    close(o, attention_want(q, k, v, scale, gate, starts), dt)
    if starts == [0, 0]:
        o = ops.attention_ex(q.to(dt).cuda(), k.to(dt).cuda(), v.to(dt).cuda(), scale)
        close(o, attention_want(q, k, v, scale, None, starts), dt)


@pytest.mark.parametrize("dt", DT)
@pytest.mark.parametrize("dh,dv", [(64, 64), (48, 80)])
def test_attention_finds_one_key_among_many(dt, dh, dv):
    """One key stands out for the last query; it is seen wherever it lies, and a later one never is."""
    from vyomai_amd import ops
    S = 300
    for where in (0, 1, 63, 64, 127, 128, 191, 255, 298, 299):
        q, k, v = rnd(1, 1, S, dh, seed=1), rnd(1, 1, S, dh, seed=2, scale=0.1), rnd(1, 1, S, dv, seed=3)
        k[0, 0, where] = q[0, 0, -1]
        o = ops.attention_ex(q.to(dt).cuda(), k.to(dt).cuda(), v.to(dt).cuda(), 1.0)
        assert torch.allclose(o[0, -1].double().cpu(), v[0, 0, where], atol=0.02), where
        if where > 0:   # the query just before it must not see it
            q2 = q.clone()
            q2[0, 0, where - 1] = q[0, 0, -1]
            o = ops.attention_ex(q2.to(dt).cuda(), k.to(dt).cuda(), v.to(dt).cuda(), 1.0)[0, where - 1].double().cpu()
            close(o, attention_want(q2[:, :, :where], k, v, 1.0, None, [0])[0, -1], dt)


def latent_want(q, uk, uv, c, n, scale, gate):
    h, dh = uk.shape[0], uk.shape[1]
    out = []
    for a in range(h):
        k, v = c[:n] @ uk[a].T, c[:n] @ uv[a].T
        s = (k @ q[a * dh:(a + 1) * dh]) * scale
        e = torch.exp(s - s.max())
        out.append((e / e.sum()) @ v)
    return torch.cat(out) * O.sigmoid(gate)


@pytest.mark.parametrize("dt", DT)
@pytest.mark.parametrize("h,dh,dv,R", [(1, 16, 8, 8), (5, 24, 40, 72), (16, 64, 88, 104), (17, 8, 72, 200), (3, 136, 128, 512),
                                       (2, 16, 24, 640), (40, 16, 16, 264)])
def test_latent_decode(dt, h, dh, dv, R):
    from vyomai_amd import ops
    lens = [1, 31, 32, 33, 64, 127, 128, 129, 300, 1000, 2, 63, 65, 96, 160, 255, 256, 257]      # keys of each sequence
    B, slots_n = len(lens), len(lens) + 2
    slots = torch.randperm(slots_n, generator=torch.Generator().manual_seed(5))[:B].to(torch.int32)
    c = rnd(slots_n, 1000, R, seed=1)
    q, gate = rnd(B, h * dh, seed=2), rnd(B, h * dv, seed=3, scale=2.0)
    uk, uv = rnd(h, dh, R, seed=4, scale=R ** -0.5), rnd(h, dv, R, seed=5, scale=R ** -0.5)
    start = torch.zeros(slots_n, dtype=torch.int32)
    cache = c.clone()
    for b, n in enumerate(lens):
        s = int(slots[b])
        start[s] = n - 1
        c[s, n // 2] = 3.0 * c[s, n // 2]                # one loud row
        cache[s] = c[s]
        cache[s, n:] = 50.0                             # whatever a slot's last owner left behind must not be seen
    scale = dh ** -0.5
    o = ops.latent_decode(q.to(dt).cuda(), uk.transpose(1, 2).contiguous().to(dt).cuda(), uv.to(dt).cuda(), cache.to(dt).cuda(),
                          start.cuda(), max(lens), scale, slots=slots.cuda(), gate=gate.to(dt).cuda())
    want = torch.stack([latent_want(q[b], uk, uv, c[int(slots[b])], n, scale, gate[b]) for b, n in enumerate(lens)])
    close(o, want, dt)
    # alone, and with a larger bound on the key count: the same up to rounding
    b = 9
    alone = ops.latent_decode(q[b:b + 1].to(dt).cuda(), uk.transpose(1, 2).contiguous().to(dt).cuda(), uv.to(dt).cuda(),
                              cache.to(dt).cuda(), start.cuda(), 1000, scale, slots=slots[b:b + 1].cuda(),
                              gate=gate[b:b + 1].to(dt).cuda())
    close(alone[0], want[b], dt)


@pytest.mark.parametrize("dt", DT)
def test_latent_decode_finds_one_key_among_many(dt):
    from vyomai_amd import ops
    n, R, dh, dv = 777, 104, 104, 32
    uk = torch.eye(R, dtype=torch.float64)[None]         # the latent is the key
    uv = rnd(1, dv, R, seed=1, scale=R ** -0.5)
    q = rnd(1, dh, seed=2)
    start = torch.tensor([n - 1], dtype=torch.int32, device="cuda")
    for where in (0, 31, 32, 127, 128, 500, 775, 776):
        c = rnd(1, n + 40, R, seed=3, scale=0.1)
        c[0, where] = q[0]
        c[0, n:] = 2 * q[0]                             # behind the newest token: invisible
        o = ops.latent_decode(q.to(dt).cuda(), uk.transpose(1, 2).contiguous().to(dt).cuda(), uv.to(dt).cuda(), c.to(dt).cuda(),
                              start, n, 1.0)
        close(o[0], uv[0] @ c[0, where], dt, 2e-2)


# ---- lightning ------------------------------------------------------------------------------------
def decay_want(p, H, dk, dv, decay, state, n):
    q, k, v = O.silu(p[:n, :H * dk]), O.silu(p[:n, H * dk:2 * H * dk]), O.silu(p[:n, 2 * H * dk:2 * H * dk + H * dv])
    outs, states = [], []
    for a in range(H):
        o, s = O.decayed_recurrence(q[:, a * dk:(a + 1) * dk], k[:, a * dk:(a + 1) * dk], v[:, a * dv:(a + 1) * dv], decay[a],
                                    state[a])
        outs.append(o)
        states.append(s)
    return torch.cat(outs, -1), torch.stack(states)


@pytest.mark.parametrize("dt", DT)
@pytest.mark.parametrize("dk,dv", [(64, 64), (8, 16), (24, 40), (128, 128), (96, 72), (136, 24), (32, 200)])
@pytest.mark.parametrize("L,count", [(1, None), (2, None), (63, None), (64, None), (65, [65, 64]), (200, [131, 200]), (130, [1, 130])])
def test_decay_attention(dt, dk, dv, L, count):
    from vyomai_amd import ops
    H, decay = 3, (0.9, 1.0, 0.0) if L < 100 else (0.999, 0.5, 0.97)
    B, slots = 2, [2, 0]
    p = rnd(B * L, H * (2 * dk + dv) + 8, seed=1)
    state = rnd(3, H, dk, dv, seed=2).float()
    start = torch.tensor([4, 9, 0], dtype=torch.int32)         # slot 2 is empty: what its last owner left is not its state
    pw = torch.tensor([[d ** i for i in range(65)] for d in decay]).float().cuda()
    sd = state.cuda()
    cnt = None if count is None else torch.tensor(count, dtype=torch.int32, device="cuda")
    o = ops.decay_attention(p.to(dt).cuda(), H, dk, dv, sd, pw, B, L, start=start.cuda(),
                            slots=torch.tensor(slots, dtype=torch.int32, device="cuda"), count=cnt).view(B, L, -1)
    for b, s in enumerate(slots):
        n = L if count is None else count[b]
        s0 = state[s].double() if start[s] > 0 else torch.zeros(H, dk, dv, dtype=torch.float64)
        want, last = decay_want(p[b * L:(b + 1) * L], H, dk, dv, decay, s0, n)
        close(o[b, :n], want, dt, 5e-5 if dt == torch.float32 else None)
        close(sd[s], last, dt, 5e-5 if dt == torch.float32 else 6e-3)
    assert torch.isfinite(o.float()).all()
    assert torch.equal(sd[1].cpu(), state[1])                  # nobody's slot


def test_chunked_state_is_32_bit():
    """Plain inputs (no activation) that bf16 holds exactly: the chunked form's state is then exact to fp32 rounding, which
    a bf16 decayed key would miss by 4e-3."""
    from vyomai_amd import ops
    H, dk, dv, L = 1, 32, 32, 256
    p = rnd(L, H * (2 * dk + dv), seed=3)
    pw = torch.tensor([[0.97 ** i for i in range(65)]]).float().cuda()
    sd = torch.zeros(1, H, dk, dv, device="cuda")
    start = torch.zeros(1, dtype=torch.int32, device="cuda")
    o = ops.decay_attention(p.to(torch.bfloat16).cuda(), H, dk, dv, sd, pw, 1, L, start=start, silu=False)
    want, last = O.decayed_recurrence(p[:, :dk], p[:, dk:2 * dk], p[:, 2 * dk:], 0.97)
    close(sd[0, 0], last, torch.bfloat16, 5e-5)
    close(o, want, torch.bfloat16, 4e-3)                       # (the output itself is stored in bf16)


@pytest.mark.parametrize("dt", DT)
def test_lightning_remembers_one_token_at_chunk_edges(dt):
    """A single loud key: every later query sees it with decay^(distance), whichever chunks the two lie in."""
    from vyomai_amd import ops
    H, dk, dv, L, d = 1, 16, 16, 260, 0.98
    pw = torch.tensor([[d ** i for i in range(65)]]).float().cuda()
    start = torch.zeros(1, dtype=torch.int32, device="cuda")
    for where in (0, 1, 62, 63, 64, 65, 127, 128, 255):
        q, k, v = torch.ones(L, dk), torch.zeros(L, dk), torch.zeros(L, dv)
        k[where], v[where] = 1.0, 1.0
        sd = torch.zeros(1, H, dk, dv, device="cuda")
        o = ops.decay_attention(torch.cat([q, k, v], -1).to(dt).cuda(), H, dk, dv, sd, pw, 1, L, start=start, silu=False)
        want = torch.tensor([dk * d ** (t - where) if t >= where else 0.0 for t in range(L)])
        err = (o[:, 0].float().cpu() - want).abs() / want.clamp(min=1.0)
        assert err.max() < (1e-5 if dt == torch.float32 else 6e-3), where


@pytest.mark.parametrize("dt", DT)
def test_silu_gated_mlp(dt):
    from vyomai_amd.layers.ffn import GatedFeedForward
    for M in (1, 3, 40):
        for width, ff in ((16, 24), (53, 35)):
            m = GatedFeedForward(width, ff).to(dt).cuda()
            w = {n: rnd(*p.shape, seed=i, scale=0.3) for i, (n, p) in enumerate(m.named_parameters())}
            with torch.no_grad():
                for n, p in m.named_parameters():
                    p.copy_(w[n])
            x = rnd(M, width, seed=9)
            y = m(pad_cols(x, up8(width)).to(dt).cuda())
            want = O.gated_mlp(x, {n.split(".")[0]: t for n, t in w.items()})
            close(y[:, :width], want, dt, None if dt == torch.float32 else 2e-2)


# ---- the model ------------------------------------------------------------------------------------
MODEL_TOL = {torch.float32: 3e-4, torch.bfloat16: 0.12}


def make(name, dt, seed=0):
    from vyomai_amd import GisitarConfig, GisitarModel
    from vyomai_amd.models.registry import load_checkpoint
    cfg = G.CONFIGS[name]
    w = G.weights(cfg, seed)
    with torch.device("meta"):
        m = GisitarModel(GisitarConfig.from_dict(cfg))
    load_checkpoint(m, w, dt, "cuda")
    return cfg, w, m.eval()


def compare(got, want, dt):
    """Root mean square over the vocabulary, of the worst position (bf16: and of the middle one)."""
    e = (got.double().cpu() - want).pow(2).mean(-1).sqrt() / want.pow(2).mean().sqrt()
    assert torch.isfinite(e).all() and e.max() < MODEL_TOL[dt], e.max()
    if dt == torch.bfloat16:
        assert e.median() < 0.04, e.median()


def run(m, ids, cuts, cache=None, slots=None):
    """Logits of every position of one sequence fed in portions (1 = the decode step)."""
    cache = cache or m.new_cache(1, 8)
    slots = slots or cache.allocate(1)
    out, at = [], 0
    for n in cuts:
        part = torch.tensor([ids[at:at + n]], device="cuda")
        if n == 1:
            out.append(m.decode(part.view(-1), cache, slots))
        else:
            out.append(m.logits(m.prefill(part, [n], cache, slots)[0]))
        at += n
    assert at == len(ids)
    return torch.cat(out)


def cut(total, size):
    return [size] * (total // size) + ([total % size] if total % size else [])


@pytest.mark.parametrize("dt", DT)
@pytest.mark.parametrize("name", list(G.CONFIGS))
def test_whole_prompt(name, dt):
    cfg, w, m = make(name, dt)
    ids = G.tokens(cfg, 150)
    lo, ref = [], []
    want = O.forward(w, cfg, ids, ref)
    c = m.new_cache()
    x = m.prefill(torch.tensor([ids], device="cuda"), [len(ids)], c, c.allocate(1), lo)
    compare(m.logits(x[0]), want, dt)
    if dt == torch.float32:
        for a, b in zip(lo, ref):
            close(a[0], b, dt, 1e-4)
    out = m(torch.tensor([ids], device="cuda"))
    compare(out.logits[0], want, dt)


@pytest.mark.parametrize("dt", DT)
@pytest.mark.parametrize("name", list(G.CONFIGS))
@pytest.mark.parametrize("cuts", ["ones", "twos", "sevens", 64, 65, "mixed"])
def test_portions_and_decoding(name, dt, cuts):
    cfg, w, m = make(name, dt)
    ids = G.tokens(cfg, 140)
    plan = {"ones": [1] * 140, "twos": [2] * 70, "sevens": [7] * 20, "mixed": [3, 1, 1, 60, 2, 1, 66, 1, 5]}.get(cuts)
    compare(run(m, ids, plan or cut(140, cuts)), O.forward(w, cfg, ids), dt)


@pytest.mark.parametrize("dt", DT)
@pytest.mark.parametrize("name", ["alternating", "odd"])
def test_unequal_batch_equals_each_alone(name, dt):
    cfg, w, m = make(name, dt)
    lens = [1, 66, 129, 2, 64, 30]
    seqs = [G.tokens(cfg, n + 8, seed=n) for n in lens]
    want = [O.forward(w, cfg, s) for s in seqs]
    cache = m.new_cache(2, 16)
    slots = cache.allocate(len(lens))
    L = max(lens)
    pad = torch.tensor([s[:n] + [0] * (L - n) for s, n in zip(seqs, lens)], device="cuda")
    x = m.prefill(pad, lens, cache, slots)
    for b, n in enumerate(lens):
        compare(m.logits(x[b, :n]), want[b][:n], dt)
    live = list(range(len(lens)))
    for t in range(8):                                     # shorter requests end earlier
        logits = m.decode(torch.tensor([seqs[b][lens[b] + t] for b in live], device="cuda"), cache, [slots[b] for b in live])
        for i, b in enumerate(live):
            compare(logits[i:i + 1], want[b][lens[b] + t:lens[b] + t + 1], dt)
        if t in (2, 5):
            cache.free([slots[live.pop(1)]])
    # a mixed continuation: portions of different lengths behind different pasts
    more = [G.tokens(cfg, n, seed=50 + n) for n in (3, 9)]
    two = live[:2]
    pad = torch.tensor([more[0] + [0] * 6, more[1]], device="cuda")
    x = m.prefill(pad, [3, 9], cache, [slots[b] for b in two])
    for i, b in enumerate(two):
        full = O.forward(w, cfg, seqs[b] + more[i])
        compare(m.logits(x[i, :len(more[i])]), full[len(seqs[b]):], dt)


@pytest.mark.parametrize("dt", DT)
def test_slots_are_used_again(dt):
    cfg, w, m = make("alternating", dt)
    cache = m.new_cache(2, 8)
    keep = cache.allocate(1)
    a, b = G.tokens(cfg, 90, seed=1), G.tokens(cfg, 40, seed=2)
    first = m.prefill(torch.tensor([a[:80]], device="cuda"), [80], cache, keep)
    for seed, n in ((3, 100), (4, 33), (5, 2), (6, 1)):    # long, then shorter owners of the same slot
        s = G.tokens(cfg, n + 3, seed=seed)
        got = cache.allocate(1)
        assert got != keep
        compare(run(m, s, ([n] if n > 1 else [1]) + [1] * 3, cache, got), O.forward(w, cfg, s), dt)
        cache.free(got)
    compare(torch.cat([m.logits(first[0]), run(m, a[80:], [1] * 10, cache, keep)]), O.forward(w, cfg, a), dt)
    del b


@pytest.mark.parametrize("dt", DT)
def test_long_decoding(dt):
    cfg, w, m = make("alternating", dt)
    ids = G.tokens(cfg, 420)
    compare(run(m, ids, [20] + [1] * 400), O.forward(w, cfg, ids), dt)


@pytest.mark.parametrize("batch", [5, 33, 70])
def test_decode_of_larger_batches(batch):
    """Batch sizes that take other product kernels (up to 4, up to 32, more rows)."""
    for dt in DT:
        cfg, w, m = make("alternating", dt)
        seqs = [G.tokens(cfg, 9, seed=100 + b) for b in range(batch)]
        cache = m.new_cache(batch, 16)
        slots = cache.allocate(batch)
        m.prefill(torch.tensor([s[:6] for s in seqs], device="cuda"), [6] * batch, cache, slots)
        for t in range(6, 9):
            logits = m.decode(torch.tensor([s[t] for s in seqs], device="cuda"), cache, slots)
        for b in (0, batch // 2, batch - 1):
            compare(logits[b:b + 1], O.forward(w, cfg, seqs[b])[-1:], dt)


# ---- entry points ---------------------------------------------------------------------------------
@pytest.mark.parametrize("name", list(G.CONFIGS))
def test_greedy_generation(name):
    cfg, w, m = make(name, torch.float32)
    prompts = [G.tokens(cfg, n, seed=n) for n in (5, 1, 12)]
    P, new = 12, 10
    ids = torch.tensor([p + [0] * (P - len(p)) for p in prompts], device="cuda")
    mask = torch.tensor([[1] * len(p) + [0] * (P - len(p)) for p in prompts], device="cuda")
    want = [O.greedy(w, cfg, p, new) for p in prompts]
    for kw in ({}, {"use_static_cache": True}, {"use_cache": False}):
        out = m.generate(ids, mask, max_len=new, **kw).cpu()
        assert out.shape == (3, P + new)
        for b, p in enumerate(prompts):
            n = len(p) + new
            assert out[b, :n].tolist() == want[b] and not out[b, n:].any(), kw


def test_generation_stops_and_samples():
    from vyomai_amd import NucleusProcessor, TopKProcessor, generate
    cfg, w, m = make("alternating", torch.float32)
    prompt = G.tokens(cfg, 6)
    ids = torch.tensor([prompt], device="cuda")
    want = O.greedy(w, cfg, prompt, 8)
    m.config.eos_token_id = want[8]                        # the third new token (or an earlier equal one)
    end = want.index(want[8], 6)
    m.config.pad_token_id = 96
    out = m.generate(ids, max_len=8).cpu()[0].tolist()
    assert out[:end + 1] == want[:end + 1] and out[end + 1:] == [96] * (14 - end - 1)
    m.config.eos_token_id = m.config.pad_token_id = None
    # top-1 sampling is greedy; the other processors stay inside the vocabulary
    assert m.generate(ids, max_len=8, processor=TopKProcessor(1.0, 1)).cpu()[0].tolist() == want
    for kw in ({"do_sample": True, "temperature": 0.8}, {"processor": NucleusProcessor(1.0, 0.9)}):
        out = m.generate(ids, max_len=8, **kw)
        assert out.shape == (1, 14) and int(out.max()) < cfg["vocab"]
    # the package's token loop
    assert generate(m, ids, max_new_tokens=8).cpu()[0].tolist() == want
    assert generate(m, ids, max_new_tokens=8, use_cache=True).cpu()[0].tolist() == want


def test_bf16_generation_follows_its_own_logits():
    cfg, _, m = make("wide", torch.bfloat16)
    prompt = G.tokens(cfg, 20)
    out = m.generate(torch.tensor([prompt], device="cuda"), max_len=12).cpu()[0].tolist()
    logits = run(m, out, [20] + [1] * 12)
    assert out[20:] == logits[19:-1].float().argmax(-1).tolist()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_replay(dtype, tmp_path):
    cfg = G.CONFIGS["odd"]
    w = G.weights(cfg)
    G.write_folder(tmp_path, cfg, w)
    a, b = G.tokens(cfg, 30, seed=1), G.tokens(cfg, 12, seed=2)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:20], "want": [0, 19]}, {"id": "b", "tokens": b[:10], "want": [9]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[20:21], "want": []}, {"id": "b", "tokens": b[10:11], "want": [0]}], "end": ["b"]},
             {"step": 2, "entries": [{"id": "a", "tokens": a[21:22], "want": []}], "end": []},
             {"step": 3, "entries": [{"id": "a", "tokens": a[22:], "want": [7]}], "end": ["a"]},
             {"step": 4, "entries": [{"id": "b", "tokens": b[:1], "want": [0]}], "end": ["b"]}]
    r = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", str(tmp_path), "--dtype", dtype,
                        "--out", str(tmp_path), "--max-tokens", "64"], input="\n".join(json.dumps(s) for s in steps) + "\n",
                       capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [l for l in r.stdout.splitlines() if l.startswith("done")] == [f"done {i}" for i in range(5)]
    fa, fb = O.forward(w, cfg, a), O.forward(w, cfg, b)
    want = {0: torch.stack([fa[0], fa[19], fb[9]]), 1: fb[10:11], 3: fa[29:30], 4: fb[:1]}
    assert {int(f.stem) for f in tmp_path.glob("*.f32")} == set(want)
    for i, t in want.items():
        got = torch.frombuffer(bytearray((tmp_path / f"{i}.f32").read_bytes()), dtype=torch.float32).view(-1, cfg["vocab"])
        assert got.shape == t.shape
        compare(got, t, torch.float32 if dtype == "float32" else torch.bfloat16)
