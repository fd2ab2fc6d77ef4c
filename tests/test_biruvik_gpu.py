"""Biruvik on the GPU: every mechanism alone and the whole model (prefill, decode, portions, unequal batches, slots used again,
window edges, far keys, generation, trace replay) against the plain oracle."""
import json
import os
import subprocess
import sys

import pytest
import torch

from oracle import biruvik_oracle as O
from tests import biruvik_cases as P

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
DT = [torch.float32, torch.bfloat16]
TOL = {torch.float32: 2e-5, torch.bfloat16: 1.2e-2}


def rnd(*shape, seed=0, scale=1.0):
    """fp64 values representable in bf16."""
    g = torch.Generator().manual_seed(seed)
    return (torch.randn(shape, generator=g) * scale).to(torch.bfloat16).double()


def close(got, want, dt, tol=None):
    got = got.double().cpu()
    err = (got - want).abs().max().item() / max(want.abs().max().item(), 1e-30)
    assert torch.isfinite(got).all() and err < (tol or TOL[dt]), err


def up8(n):
    return (n + 7) // 8 * 8


def pad_cols(t, n):
    out = torch.zeros(*t.shape[:-1], n, dtype=t.dtype)
    out[..., : t.shape[-1]] = t
    return out


def i32(values):
    return torch.tensor(values, dtype=torch.int32, device="cuda")


def rounded(t, dt):
    return t.to(torch.bfloat16).double() if dt == torch.bfloat16 else t


def pack(rows, *parts):
    """True-width rows (M, .) of parts (heads, columns each) side by side -> every head padded by itself."""
    M, out, at = rows.shape[0], [], 0
    for n, d in parts:
        out.append(pad_cols(rows[:, at: at + n * d].reshape(M, n, d), up8(d)).view(M, -1))
        at += n * d
    return torch.cat(out, 1)


def head_vector(w, n):
    return pad_cols(w.view(n, -1), up8(w.numel() // n)).view(-1).float().cuda()


# ---- norms, products ------------------------------------------------------------------------------
@pytest.mark.parametrize("dt", DT)
@pytest.mark.parametrize("heads,dim", [(3, 5), (1, 8), (7, 24), (4, 64), (16, 128), (2, 232), (1, 600)])
def test_head_norm_with_a_shared_weight(dt, heads, dim):
    from vyomai_amd import ops
    M, NP, eps = 37, up8(dim), 1e-2
    x = rounded(rnd(M, heads, dim, seed=1) * torch.logspace(-2, 2, heads)[:, None].double(), torch.bfloat16)
    w = 1 + 0.5 * rnd(dim, seed=2)
    out = ops.head_norm_gate(pad_cols(x, NP).view(M, -1).to(dt).cuda(), heads, dim, None, eps, w=head_vector(w, 1)).view(M, heads, NP)
    close(out[..., :dim], O.rms(x, eps) * w, dt)
    assert not out[..., dim:].any()


@pytest.mark.parametrize("dt", DT)
@pytest.mark.parametrize("N,K", [(40, 24), (3000, 256), (96, 2048), (264, 6144)])
@pytest.mark.parametrize("M", [1, 3, 20, 70, 300, 2000])
def test_products_with_squared_relu_capped_logits_and_bias(dt, M, N, K):
    from vyomai_amd import ops
    from vyomai_amd._lib import ACT_RELU2
    x, w, b = rnd(M, K, seed=1), rnd(N, K, seed=2, scale=K ** -0.5), rnd(N, seed=3)
    xd, wd = x.to(dt).cuda(), w.to(dt).cuda()
    z = x @ w.T
    close(ops.linear(xd, wd, act=ACT_RELU2), torch.clamp(z, min=0) ** 2, dt)
    close(ops.linear(xd, wd, b.to(dt).cuda()), z + b, dt)
    for cap in (0.7, 30.0):
        y = ops.linear_softcap(xd, wd, cap)
        close(y, O.softcap(z, cap), dt)
        assert float(y.abs().max()) <= cap * (1 + 2 ** -7)


# ---- queries, keys, values ------------------------------------------------------------------------
@pytest.mark.parametrize("dt", DT)
@pytest.mark.parametrize("h,hk,dim,vdim", [(4, 2, 16, 24), (3, 1, 10, 13), (16, 4, 64, 128), (40, 8, 8, 64), (1, 1, 250, 40), (2, 2, 136, 8)])
@pytest.mark.parametrize("B,L", [(2, 5), (1, 700)])
def test_head_norms_temperature_and_cache_rows(dt, h, hk, dim, vdim, B, L):
    """Norms over single maps of single heads; queries times their temperature; keys and values in their cache rows."""
    from vyomai_amd import ops
    eps, coef, every, dp, vp = 1e-2, 0.8, 13, up8(dim), up8(vdim)
    q, k, v = rnd(B * L, h, 2, dim, seed=1, scale=3.0), rnd(B * L, hk, 2, dim, seed=2, scale=0.3), rnd(B * L, hk, vdim, seed=3)
    q *= torch.logspace(-1, 1, 2 * h).view(h, 2, 1).double()
    q = rounded(q, torch.bfloat16)
    wq, wk = 1 + 0.3 * rnd(dim, seed=4), 1 + 0.3 * rnd(dim, seed=5)
    p = pack(torch.cat([q.flatten(1), k.flatten(1), v.flatten(1)], 1), (2 * h, dim), (2 * hk, dim), (hk, vdim)).to(dt).cuda()
    first, slots = [300, 0][:B], [2, 1][:B]
    start = torch.zeros(3, dtype=torch.int32, device="cuda")
    start[slots] = i32(first)
    counts = [L, 3][:B]
    ring = torch.full((3, hk, first[0] + L, 2 * dp + vp), 77.0, dtype=dt, device="cuda")
    prep = ops.QkvPrep(head_vector(wq, 1).repeat(2 * h), head_vector(wk, 1).repeat(2 * hk), dim, dim, eps, group=dp, temp_every=every, temp_coef=coef)
    nk, gk = 2 * h * dp, 2 * hk * dp
    ops.qkv_rows(p, B, L, h, hk, 2 * dp, vp, 0, nk, nk + gk, prep, ring=ring, slots=i32(slots), start=start, count=i32(counts))
    tol = 2e-5 if dt == torch.float32 else 5e-3
    for b in range(B):
        part = slice(b * L, (b + 1) * L)
        temp = torch.tensor([O.temperature(first[b] + i, coef, every) for i in range(L)], dtype=torch.float64)
        wantq, wantk = O.rms(q[part], eps) * wq * temp[:, None, None, None], O.rms(k[part], eps) * wk
        got = p[part]
        close(got[:, :nk].view(L, h, 2, dp)[..., :dim], wantq, dt, tol)
        close(got[:, nk: nk + gk].view(L, hk, 2, dp)[..., :dim], wantk, dt, tol)
        n = counts[b]
        rows = ring[slots[b], :, first[b]: first[b] + n].transpose(0, 1)
        close(rows[..., : 2 * dp].unflatten(-1, (2, dp))[..., :dim], wantk[:n], dt, tol)
        assert torch.equal(rows[..., 2 * dp:][..., :vdim].double().cpu(), v[part][:n])
        assert bool((ring[slots[b], :, : first[b]] == 77).all()) and bool((ring[slots[b], :, first[b] + n:] == 77).all())
    assert bool((ring[0] == 77).all())


@pytest.mark.parametrize("dt", DT)
def test_head_norms_with_rotary_positions(dt):
    """The same kernels with one map per head, rotated, in windowed attention: prompt rows and a decode step."""
    from oracle import padulorn_oracle as PO
    from vyomai_amd import ops
    from vyomai_amd.layers.positional_embeddings import PairRotary
    h, hk, dim, vdim, eps, T, window = 4, 2, 24, 16, 1e-3, 40, 17
    rot = {"base": 90.0, "dims": 10}
    table = PairRotary(rot["base"], rot["dims"]).table(T, "cuda")
    rows, wq, wk = rnd(T, (h + hk) * dim + hk * vdim, seed=1), 1 + 0.3 * rnd(dim, seed=2), 1 + 0.3 * rnd(dim, seed=3)
    q = O.rms(rows[:, : h * dim].view(T, h, dim), eps) * wq
    k = O.rms(rows[:, h * dim:(h + hk) * dim].view(T, hk, dim), eps) * wk
    q, k = (rounded(torch.stack([PO.rotate(t[:, a], rot, "pairs") for a in range(t.shape[1])], 1), dt) for t in (q, k))
    v = rows[:, (h + hk) * dim:].view(T, hk, vdim)
    prep = ops.QkvPrep(wq.repeat(h).float().cuda(), wk.repeat(hk).float().cuda(), dim, dim, eps, group=dim)
    p, at = rows.to(dt).cuda(), dict(start=torch.zeros(1, dtype=torch.int32, device="cuda"))
    ring = torch.zeros(1, hk, window, dim + vdim, dtype=dt, device="cuda")
    n = T - 3
    first = p[:n].clone()
    ops.qkv_rows(first, 1, n, h, hk, dim, vdim, 0, h * dim, (h + hk) * dim, prep, rotary=table, ring=ring, **at)
    close(first[:, : h * dim].view(n, h, dim), q[:n], dt, None if dt == torch.float32 else 5e-3)
    at["start"] += n
    for t in range(n, T):
        o = ops.window_decode(p[t:t + 1].clone(), h, hk, dim, vdim, ring, 0.3, at["start"], t + 1, rotary=table, prep=prep)
        at["start"] += 1
        want = torch.cat([PO.window_attention(q[:, a], k[:, a // 2], v[:, a // 2], 0.3, window, 0)[t] for a in range(h)])
        close(o[0], want, dt)


# ---- differential attention -----------------------------------------------------------------------
class Diff:
    """B sequences through the calls of layers/differential_attention.py, slots out of order, old garbage in the cache."""
    eps = 1e-3

    def __init__(self, dt, h, hk, dim, vdim, B, rows, lam=0.55, out_scale=0.7, coef=0.5, every=11, spread=2.0):
        self.dt, self.h, self.hk, self.dim, self.vdim, self.B, self.spread = dt, h, hk, dim, vdim, B, spread
        self.lam, self.out_scale, self.coef, self.every = lam, out_scale, coef, every
        self.slots = [2 * b + 1 for b in reversed(range(B))]
        dp, vp = up8(dim), up8(vdim)
        self.ring = torch.full((2 * B + 1, hk, rows, 2 * dp + vp), float("nan"), dtype=dt, device="cuda")
        self.start = torch.zeros(2 * B + 1, dtype=torch.int32, device="cuda")
        self.past = [torch.zeros(0, self.width, dtype=torch.float64) for _ in range(B)]
        self.wq, self.wk = spread * (1 + 0.3 * rnd(dim, seed=3)), 1 + 0.3 * rnd(dim, seed=4)
        self.seed = 10

    @property
    def width(self):
        return 2 * (self.h + self.hk) * self.dim + self.hk * self.vdim

    def fresh(self, counts, rows=None):
        from vyomai_amd import _lib, ops
        self.seed += 1
        L, dp = max(counts), up8(self.dim)
        rows = rnd(self.B, L, self.width, seed=self.seed) if rows is None else rows
        for b, n in enumerate(counts):
            self.past[b] = torch.cat([self.past[b], rows[b, :n]])
        p = pack(rows.reshape(self.B * L, -1), (2 * self.h, self.dim), (2 * self.hk, self.dim), (self.hk, self.vdim)).to(self.dt).cuda()
        prep = ops.QkvPrep(head_vector(self.wq, 1).repeat(2 * self.h), head_vector(self.wk, 1).repeat(2 * self.hk), self.dim, self.dim, self.eps,
                           group=dp, temp_every=self.every, temp_coef=self.coef)
        return p, L, prep, _lib.VyDiff(self.lam, self.out_scale, self.eps, self.vdim)

    def want(self, b, last):
        """Outputs of the last `last` tokens of sequence b."""
        x, T, h, hk, dim = self.past[b], self.past[b].shape[0], self.h, self.hk, self.dim
        q = O.rms(x[:, : 2 * h * dim].view(T, h, 2, dim), self.eps) * self.wq
        temp = torch.tensor([O.temperature(i, self.coef, self.every) if self.every else 1.0 for i in range(T)], dtype=torch.float64)
        q = rounded(q * temp[:, None, None, None], self.dt)
        k = rounded(O.rms(x[:, 2 * h * dim: 2 * (h + hk) * dim].view(T, hk, 2, dim), self.eps) * self.wk, self.dt)
        v = x[:, 2 * (h + hk) * dim:].view(T, hk, self.vdim)
        i = torch.arange(T - last, T)
        out = []
        for a in range(h):
            g = a // (h // hk)
            s = [(q[T - last:, a, m] @ k[:, g, m].T * dim ** -0.5).masked_fill(torch.arange(T)[None] > i[:, None], float("-inf")).softmax(-1) @ v[:, g]
                 for m in (0, 1)]
            out.append(O.differential_head(s[0], s[1], torch.tensor(self.lam), 1 - self.out_scale, self.eps))
        return torch.cat(out, -1)

    def got(self, o):
        o = o.unflatten(-1, (self.h, up8(self.vdim)))
        assert not o[..., self.vdim:].any()
        return o[..., : self.vdim].flatten(-2)

    def prefill(self, counts, rows=None):
        from vyomai_amd import ops
        p, L, prep, diff = self.fresh(counts, rows)
        dim, vdim, h, hk = 2 * up8(self.dim), up8(self.vdim), self.h, self.hk
        at = dict(slots=i32(self.slots), start=self.start, count=i32(counts) if len(set(counts)) > 1 else None)
        ops.qkv_rows(p, self.B, L, h, hk, dim, vdim, 0, h * dim, (h + hk) * dim, prep, ring=self.ring, **at)
        o = ops.diff_attention(p, self.B, L, h, hk, dim, vdim, self.ring, self.dim ** -0.5, diff, **at)
        assert torch.isfinite(o).all()                       # (the padding too)
        self.start[self.slots] += i32(counts)
        return self.got(o.view(self.B, L, -1))

    def decode(self, rows=None):
        from vyomai_amd import ops
        p, _, prep, diff = self.fresh([1] * self.B, rows)
        top = max(x.shape[0] for x in self.past)
        o = ops.window_decode(p, self.h, self.hk, 2 * up8(self.dim), up8(self.vdim), self.ring, self.dim ** -0.5, self.start, top, prep=prep,
                              diff=diff, slots=i32(self.slots))
        self.start[self.slots] += 1
        return self.got(o)


SHAPES = [(6, 2, 32, 64), (2, 1, 64, 128), (3, 3, 10, 13), (6, 2, 16, 40), (40, 2, 8, 24), (2, 1, 72, 200), (2, 2, 136, 64), (1, 1, 250, 250),
          (4, 1, 24, 64), (2, 2, 61, 125), (2, 1, 264, 16)]


@pytest.mark.parametrize("dt", DT)
@pytest.mark.parametrize("h,hk,dim,vdim", SHAPES)
def test_differential_attention(dt, h, hk, dim, vdim):
    """Prompts, portions down to two tokens behind a past, unequal counts, decoding in between."""
    d = Diff(dt, h, hk, dim, vdim, 3, 420)
    for counts in ([200, 1, 65], [2, 2, 2], [3, 90, 1], None, [130, 64, 128], None, None):
        o = d.decode()[:, None] if counts is None else d.prefill(counts)
        for b, n in enumerate(counts or [1, 1, 1]):
            close(o[b, :n], d.want(b, n), dt)
    untouched = [s for s in range(7) if s not in d.slots]
    assert torch.isnan(d.ring[untouched]).all()


@pytest.mark.parametrize("dt", DT)
@pytest.mark.parametrize("dim,vdim", [(32, 64), (64, 128), (16, 40)])
def test_differential_decoding_over_a_long_context(dt, dim, vdim):
    """The context is cut into slices that a second launch puts together."""
    d = Diff(dt, 5, 1, dim, vdim, 2, 1700)
    d.prefill([1600, 3])
    for _ in range(3):
        o = d.decode()
    for b in range(2):
        close(o[b:b + 1], d.want(b, 1), dt)


@pytest.mark.parametrize("dt", DT)
@pytest.mark.parametrize("dim,vdim", [(32, 64), (64, 128), (24, 40)])
@pytest.mark.parametrize("how", ["prompt", "decoding"])
def test_differential_attention_finds_a_far_key(dt, dim, vdim, how):
    """One query points at one key hundreds of tokens back, on one map only; at the token itself; at the next one, which it must
    not see."""
    T, lam = 500, 0.25
    for far in (0, 5, 63, 64, 65, 255, 256, T - 2, T - 1):
        for m in (0, 1):
            d = Diff(dt, 1, 1, dim, vdim, 1, T + 1, lam=lam, spread=6.0, every=0)
            rows = rnd(1, T + 1, d.width, seed=1)
            aim = rnd(dim, seed=2)
            rows[0, T - 1, m * dim:(m + 1) * dim] = aim / d.wq * d.wk.abs().max()
            rows[0, far, (2 + m) * dim:(3 + m) * dim] = aim / d.wk
            rows[0, T, (2 + m) * dim:(3 + m) * dim] = 4 * aim / d.wk
            rows = rounded(rows, torch.bfloat16)
            if how == "prompt":
                o = d.prefill([T + 1], rows)[0, T - 1]
                want = d.want(0, 2)[0]
            else:
                d.prefill([T - 1], rows[:, : T - 1])
                o, want = d.decode(rows[:, T - 1:T])[0], d.want(0, 1)[0]
            close(o, want, dt)
            v = rows[0, far, 4 * dim:]
            other = O.rms(v if m == 0 else -v, 0.0)
            alike = torch.nn.functional.cosine_similarity(o.double().cpu(), other, dim=0)
            assert m == 1 or alike > 0.9, (far, alike)


@pytest.mark.parametrize("dt", DT)
def test_temperature_steps(dt):
    """Each position's own factor, in prompts, portions and decoding, at the places where it steps."""
    d = Diff(dt, 2, 1, 16, 32, 1, 64, coef=3.0, every=8)
    o = [d.prefill([7])[0]] + [d.decode() for _ in range(3)] + [d.prefill([5])[0], d.prefill([2])[0]] + [d.decode() for _ in range(16)]
    close(torch.cat([x.view(-1, x.shape[-1]) for x in o]), d.want(0, 33), dt)


# ---- gated linear attention -----------------------------------------------------------------------
def gated(rows, h, dim, vdim, bias, lower, states=None):
    """Oracle on true-width rows (T, [q | z | v]) -> (T, h * vdim), states."""
    S = states or [torch.zeros(dim, vdim, dtype=torch.float64) for _ in range(h)]
    q, v = O.silu(rows[:, : h * dim]), rows[:, 2 * h * dim:]
    f = O.forget(rows[:, h * dim: 2 * h * dim] + bias, lower)
    out = [O.recurrence(q[:, a * dim:(a + 1) * dim], f[:, a * dim:(a + 1) * dim], v[:, a * vdim:(a + 1) * vdim], S[a]) for a in range(h)]
    return torch.cat(out, -1), S


def run_gated(dt, rows, h, dim, vdim, bias, lower, state, slots, start, counts):
    from vyomai_amd import ops
    B, L = rows.shape[:2]
    p = pack(rows.reshape(B * L, -1), (h, dim), (h, dim), (h, vdim)).to(dt).cuda()
    low = 1.0 - head_vector(1.0 - lower, h)
    o = ops.gated_attention(p, h, up8(dim), up8(vdim), state, low, head_vector(bias, h), B, L, start=start, slots=i32(slots),
                            count=i32(counts) if len(set(counts)) > 1 else None)
    start[slots] += i32(counts)
    return o.view(B, L, h, up8(vdim))


GATES = {"mixed": (2.0, 2.5, True), "open": (9.0, 1.0, False), "closed": (-12.0, 4.0, False), "extreme": (0.0, 30.0, False)}


@pytest.mark.parametrize("dt", DT)
@pytest.mark.parametrize("gates", list(GATES))
@pytest.mark.parametrize("h,dim,vdim", [(2, 16, 24), (3, 10, 13), (1, 64, 72), (2, 128, 128), (2, 40, 8), (1, 136, 16), (1, 24, 200), (1, 512, 8)])
@pytest.mark.parametrize("portions", [[200], [2, 63, 1, 64, 1, 65], [1, 1, 1, 130, 2]])
def test_gated_linear_attention(dt, gates, h, dim, vdim, portions):
    """Gates between 0 (to the last bit) and 1, portions around chunk and block borders, unequal counts, garbage in empty slots."""
    at, spread, low = GATES[gates]
    B, slots = 2, [3, 1]
    bias = rnd(h * dim, seed=50, scale=spread) + at
    lower = (torch.rand(h * dim, generator=torch.Generator().manual_seed(51)).double() - 0.3).clamp(min=0.0) * low
    bias, lower = rounded(bias, torch.bfloat16), rounded(lower, torch.bfloat16)
    state = torch.full((4, h, up8(dim), up8(vdim)), float("nan"), device="cuda")
    start = torch.zeros(4, dtype=torch.int32, device="cuda")
    past = [None, None]
    for i, L in enumerate(portions):
        counts = [L, max(1, L - 30)]
        rows = rnd(B, L, 2 * h * dim + h * vdim, seed=i)
        o = run_gated(dt, rows, h, dim, vdim, bias, lower, state, slots, start, counts)
        assert torch.isfinite(o).all() and not o[..., vdim:].any()
        for b, c in enumerate(counts):
            want, past[b] = gated(rows[b, :c], h, dim, vdim, bias, lower, past[b])
            close(o[b, :c, :, :vdim].flatten(-2), want, dt, None if dt == torch.float32 else 5e-3)
            close(state[slots[b], :, :dim, :vdim], torch.stack(past[b]), dt, None if dt == torch.float32 else 1e-4)
    assert torch.isnan(state[[0, 2]]).all() and not state[slots][:, :, dim:].any() and not state[slots][..., vdim:].any()


@pytest.mark.parametrize("dt", DT)
@pytest.mark.parametrize("dim", [24, 128])
def test_gated_linear_attention_keeps_and_forgets(dt, dim):
    """A value written hundreds of tokens back through a gate that is open for it alone, found by the query that reads its channel;
    the channels whose gates closed since then hold nothing of it."""
    T, far = 400, 5
    bias, lower = torch.full((dim,), 14.0, dtype=torch.float64), torch.zeros(dim, dtype=torch.float64)
    rows = torch.zeros(T, 2 * dim + dim, dtype=torch.float64)
    rows[:, : dim] = -30.0                                       # queries of about 0 ...
    loud = rnd(dim, seed=1, scale=3.0)
    rows[:, 2 * dim:] = rnd(T, dim, seed=2, scale=0.05)
    rows[far, 2 * dim:] = loud
    rows[far, dim:dim + 2] = -14.0                               # channels 0 and 1 are written at this token
    rows[200, dim + 1] = -40.0                                   # channel 1 forgets on the way
    for t, c in ((390, 0), (391, 1), (T - 2, 0), (T - 1, 1)):
        rows[t, c] = 10.0                                        # ... but for one channel (two in the prompt, two decoded)
    state, start = torch.zeros(1, 1, dim, dim, device="cuda"), torch.zeros(1, dtype=torch.int32, device="cuda")
    got = []
    for a, b in [(0, T - 5)] + [(t, t + 1) for t in range(T - 5, T)]:
        got.append(run_gated(dt, rows[None, a:b], 1, dim, dim, bias, lower, state, [0], start, [b - a])[0, :, 0])
    got = torch.cat(got).double().cpu()
    want, _ = gated(rows, 1, dim, dim, bias, lower)
    for t, c in ((390, 0), (391, 1), (T - 2, 0), (T - 1, 1)):
        alike = torch.nn.functional.cosine_similarity(got[t], loud, dim=0)
        assert (alike > 0.99) if c == 0 else (alike.abs() < 0.9), (t, alike)
        close(got[t], want[t], dt, None if dt == torch.float32 else 5e-3)


# ---- windowed latent attention --------------------------------------------------------------------
def latent_layer(dt, cfg, width, eps, seed=0, **kw):
    from vyomai_amd.layers.latent_attention import LatentAttention
    m = LatentAttention(width, cfg["heads"], cfg["dim"], cfg["vdim"], None, cfg["kv_rank"], cfg["scale"], eps, window=cfg["mask"]["size"],
                        head_gate=True, **kw).to(dt).cuda()
    names = {"q": "query.weight", "dkv": "kv_down.weight", "dkv.norm": "kv_norm.weight", "uk": "k_up.weight", "uv": "v_up.weight", "g": "gate.weight",
             "o": "out.weight"}
    par, w = dict(m.named_parameters()), {}
    with torch.no_grad():
        for i, (short, long) in enumerate(names.items()):
            t = par[long]
            w[short] = rnd(*t.shape, seed=seed + i, scale=1.5 * t.shape[-1] ** -0.5) if t.dim() == 2 else 1 + 0.2 * rnd(*t.shape, seed=seed + i)
            w[short] = rounded(w[short], torch.bfloat16)
            t.copy_(w[short])
    return m.requires_grad_(False), w


class Mixer:
    """One mixer over a cache of its own: portions of B sequences (prefill) and single tokens through a decode plan's kernels."""

    def __init__(self, m, dt, width, B, capacity=8):
        from vyomai_amd import SlotCache
        self.m, self.dt, self.width, self.B = m, dt, width, B
        self.cache = SlotCache([m.cache_spec()], dt, "cuda", 2 * B, capacity)
        self.slots = self.cache.allocate(B)

    def prefill(self, rows, counts):
        L = rows.shape[1]
        batch = self.cache.reserve(self.slots, counts)
        h = pad_cols(rows.reshape(self.B * L, -1), up8(self.width)).to(self.dt).cuda()
        y = self.m(h, self.B, L, batch, 0).view(self.B, L, -1)[..., : self.width]
        self.cache.advance(self.slots, counts)
        return y

    def decode(self, rows):
        from vyomai_amd import ops
        m, p, batch = self.m, self.m.packed(), self.cache.reserve(self.slots, [1] * self.B)
        x = ops.linear(pad_cols(rows, up8(self.width)).to(self.dt).cuda(), p.w_in)
        ring, kr = self.cache.buffers[0], p.c_norm.numel()
        ops.latent_norm(x, None, p.n_first, p.c_norm, m.kv_rank, self.B, 1, m.eps, cache=ring, slots=batch.slots, start=batch.start, want_c=False)
        o = ops.latent_decode(x[:, : p.n_first], p.w_ukt, p.w_uv.view(m.heads, -1, kr), ring, batch.start, batch.max_keys, m.scale,
                              slots=batch.slots, gate=x[:, p.n_first + kr:], gate_heads=True)
        self.cache.advance(self.slots, [1] * self.B)
        return ops.linear(o, p.w_o)[:, : self.width]


LATENTS = [(4, 16, 24, 32, 24), (3, 10, 13, 19, 1), (17, 8, 40, 64, 2), (2, 64, 64, 128, 64), (2, 128, 128, 256, 33), (1, 24, 72, 520, 65),
           (5, 136, 8, 40, 130)]


@pytest.mark.parametrize("dt", DT)
@pytest.mark.parametrize("heads,dim,vdim,kv_rank,window", LATENTS)
def test_windowed_latent_attention(dt, heads, dim, vdim, kv_rank, window):
    cfg, width, eps, B = P.latent(heads, dim, vdim, kv_rank, window)["mixer"], 44, 1e-3, 3
    m, w = latent_layer(dt, cfg, width, eps)
    run = Mixer(m, dt, width, B)
    past = [torch.zeros(0, width, dtype=torch.float64) for _ in range(B)]
    for i, counts in enumerate(([70, 1, 30], None, [2, 2, 2], [1, 140, 33], None, None, [64, 3, 1], None)):
        n = counts or [1] * B
        rows = rnd(B, max(n), width, seed=100 + i)
        o = run.decode(rows[:, 0])[:, None] if counts is None else run.prefill(rows, counts)
        for b in range(B):
            past[b] = torch.cat([past[b], rows[b, : n[b]]])
            close(o[b, : n[b]], O.latent_attention(past[b], w, cfg, eps)[-n[b]:], dt, None if dt == torch.float32 else 3e-2)
    assert run.cache.buffers[0].shape[2] == min(window, run.cache.capacity)


@pytest.mark.parametrize("dt", DT)
@pytest.mark.parametrize("kv_rank", [64, 256])
@pytest.mark.parametrize("window", [1, 2, 31, 32, 33, 64, 100])
@pytest.mark.parametrize("how", ["prompt", "portions", "decoding"])
def test_edges_of_the_latent_window(dt, kv_rank, window, how):
    """A loud token is seen as the window's last one, and not a token further."""
    T, width, eps = 130, kv_rank, 1e-6
    cfg = P.latent(1, kv_rank, kv_rank, kv_rank, window, scale=1.0)["mixer"]
    m, w = latent_layer(dt, cfg, width, eps)
    eye = torch.eye(kv_rank, dtype=torch.float64)
    with torch.no_grad():                                       # keys and values are the normed tokens themselves, queries shifted ones
        for name, t in (("q", m.query), ("dkv", m.kv_down), ("uk", m.k_up), ("uv", m.v_up), ("o", m.out)):
            w[name] = eye.roll(1, 0) if name == "q" else eye
            t.weight.copy_(w[name])
        w["dkv.norm"], w["g"] = torch.ones(kv_rank, dtype=torch.float64), torch.zeros(1, kv_rank, dtype=torch.float64)
        m.kv_norm.weight.fill_(1.0)
        m.gate.weight.zero_()
    for where, seen in ((T - window, True), (T - 1 - window, False)):
        rows = rnd(1, T, width, seed=1, scale=0.1)
        loud = rnd(width, seed=2)
        rows[0, where] = loud
        if where != T - 1:
            rows[0, -1] = loud.roll(-1) * 0.5                   # (its query points at the loud token, its own key does not)
        run = Mixer(m, dt, width, 1)
        if how == "prompt":
            o = run.prefill(rows, [T])[0, -1]
        elif how == "portions":
            run.prefill(rows[:, :50], [50])
            run.prefill(rows[:, 50:T - 2], [T - 52])
            o = run.prefill(rows[:, T - 2:], [2])[0, -1]
        else:
            run.prefill(rows[:, :40], [40])
            for t in range(40, T):
                o = run.decode(rows[:, t])[0]
        want = O.latent_attention(rows[0], w, cfg, eps)[-1]
        close(o, want, dt, None if dt == torch.float32 else 2e-2)
        if window > 1:
            gone = rows.clone()
            gone[0, where] = -loud
            changes = (O.latent_attention(gone[0], w, cfg, eps)[-1] - want).abs().max() > 0.1
            assert bool(changes) == seen


# ---- the model ------------------------------------------------------------------------------------
MODEL_TOL = {torch.float32: (3e-4, 3e-5), torch.bfloat16: (0.3, 0.03)}   # worst and middle position (bf16: rounding the oracle's
# products alone moves single positions by 0.15, where a norm divides by little)


def make(name, dt, seed=0):
    from vyomai_amd import BiruvikConfig, BiruvikModel
    from vyomai_amd.models.registry import load_checkpoint
    cfg = P.CONFIGS[name] if isinstance(name, str) else name
    w = P.weights(cfg, seed)
    with torch.device("meta"):
        m = BiruvikModel(BiruvikConfig.from_dict(cfg))
    load_checkpoint(m, w, dt, "cuda")
    return cfg, w, m.eval()


def compare(got, want, dt):
    """Root mean square over the vocabulary, every position."""
    e = (got.double().cpu() - want).pow(2).mean(-1).sqrt() / want.pow(2).mean().sqrt()
    assert torch.isfinite(e).all() and e.max() < MODEL_TOL[dt][0] and e.median() < MODEL_TOL[dt][1], (e.max(), e.median())


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


_REF = {}


def reference(name, ids, seed=0):
    key = name, tuple(ids), seed
    if key not in _REF:
        lo = []
        cfg = P.CONFIGS[name]
        _REF[key] = O.forward(P.weights(cfg, seed), cfg, ids, lo), lo
    return _REF[key]


@pytest.mark.parametrize("dt", DT)
@pytest.mark.parametrize("name", list(P.CONFIGS))
def test_whole_prompt(name, dt):
    cfg, w, m = make(name, dt)
    ids = P.tokens(cfg, 140)
    want, ref = reference(name, ids)
    lo = []
    c = m.new_cache()
    x = m.prefill(torch.tensor([ids], device="cuda"), [len(ids)], c, c.allocate(1), lo)
    compare(m.logits(x[0]), want, dt)
    if dt == torch.float32:
        for a, b in zip(lo, ref):
            close(a[0], b, dt, 1e-4)
    compare(m(torch.tensor([ids], device="cuda")).logits[0], want, dt)


@pytest.mark.parametrize("dt", DT)
@pytest.mark.parametrize("name", list(P.CONFIGS))
@pytest.mark.parametrize("cuts", ["ones", "twos", "sevens", "sixties", "mixed"])
def test_portions_and_decoding(name, dt, cuts):
    cfg, w, m = make(name, dt)
    ids = P.tokens(cfg, 140)
    plan = {"ones": [1] * 140, "twos": [2] * 70, "sevens": [7] * 20, "sixties": [65, 64, 11], "mixed": [3, 1, 1, 60, 2, 1, 66, 1, 5]}[cuts]
    compare(run(m, ids, plan), reference(name, ids)[0], dt)


@pytest.mark.parametrize("dt", DT)
@pytest.mark.parametrize("name", ["plain", "odd"])
def test_unequal_batch_equals_each_alone(name, dt):
    cfg, w, m = make(name, dt)
    lens = [1, 66, 129, 2, 64, 30]
    seqs = [P.tokens(cfg, n + 8, seed=n) for n in lens]
    want = [reference(name, s)[0] for s in seqs]
    cache = m.new_cache(2, 16)
    slots = cache.allocate(len(lens))
    L = max(lens)
    pad = torch.tensor([s[:n] + [0] * (L - n) for s, n in zip(seqs, lens)], device="cuda")
    x = m.prefill(pad, lens, cache, slots)
    assert torch.isfinite(x).all()
    pairs = [(m.logits(x[b, :n]), want[b][:n]) for b, n in enumerate(lens)]
    live = list(range(len(lens)))
    steps = {b: [] for b in live}
    for t in range(8):                                     # shorter requests end earlier
        logits = m.decode(torch.tensor([seqs[b][lens[b] + t] for b in live], device="cuda"), cache, [slots[b] for b in live])
        for i, b in enumerate(live):
            steps[b].append(logits[i:i + 1])
        if t in (2, 5):
            cache.free([slots[live.pop(1)]])
    for b, rows in steps.items():
        pairs.append((torch.cat(rows), want[b][lens[b]:lens[b] + len(rows)]))
    # a mixed continuation: portions of different lengths behind different pasts
    more = [P.tokens(cfg, n, seed=50 + n) for n in (3, 9)]
    pad = torch.tensor([more[0] + [0] * 6, more[1]], device="cuda")
    x = m.prefill(pad, [3, 9], cache, [slots[b] for b in live[:2]])
    for i, b in enumerate(live[:2]):
        full = O.forward(w, cfg, seqs[b] + more[i])
        pairs.append((m.logits(x[i, :len(more[i])]), full[len(seqs[b]):]))
    compare(torch.cat([a for a, _ in pairs]), torch.cat([b for _, b in pairs]), dt)


@pytest.mark.parametrize("dt", DT)
def test_slots_are_used_again(dt):
    cfg, w, m = make("plain", dt)
    cache = m.new_cache(2, 8)
    keep = cache.allocate(1)
    a = P.tokens(cfg, 90, seed=1)
    first = m.prefill(torch.tensor([a[:80]], device="cuda"), [80], cache, keep)
    for seed, n in ((3, 100), (4, 33), (5, 2), (6, 1)):    # long, then shorter owners of the same slot
        s = P.tokens(cfg, n + 3, seed=seed)
        got = cache.allocate(1)
        assert got != keep
        compare(run(m, s, [n, 1, 1, 1], cache, got), reference("plain", s)[0], dt)
        for buf in cache.buffers:                          # whatever the owner leaves behind
            buf[got] = float("nan")
        cache.free(got)
    compare(torch.cat([m.logits(first[0]), run(m, a[80:], [1] * 10, cache, keep)]), reference("plain", a)[0], dt)


@pytest.mark.parametrize("dt", DT)
def test_long_decoding(dt):
    cfg, w, m = make("odd", dt)
    ids = P.tokens(cfg, 330)
    cache = m.new_cache(1, 8)
    compare(run(m, ids, [20] + [1] * 310, cache, cache.allocate(1)), reference("odd", ids)[0], dt)
    assert [cache.buffers[i].shape[2] for i in (2, 4)] == [30, 19]       # no ring outgrows its window


@pytest.mark.parametrize("dt", DT)
@pytest.mark.parametrize("how", ["prompt", "decoding"])
def test_a_layer_sees_its_window_and_no_further(dt, how):
    """Latent layers alone: changing the window's first token changes the last logits, changing the one before it does not; a
    differential layer sees every token."""
    for window in (1, 5, 32, 64, 99):
        cfg = P.config([P.latent(2, 16, 16, 24, window, mlp=P.dense(16))])
        _, _, m = make(cfg, dt)
        ids = P.tokens(cfg, 100)

        def last(s):
            return run(m, s, [100] if how == "prompt" else [60] + [1] * 40)[-1].float()
        base = last(ids)
        for at, seen in ((100 - window, True), (99 - window, False)):
            if at >= 0:
                other = list(ids)
                other[at] = (other[at] + 1) % cfg["vocab"]
                assert torch.equal(last(other), base) != seen, (window, at)
    cfg = P.config([P.attention(2, 1, 16, 16)])
    _, _, m = make(cfg, torch.float32)
    ids = P.tokens(cfg, 100)
    base = last(ids)
    for at in (0, 1, 36, 63, 98):
        other = list(ids)
        other[at] = (other[at] + 1) % cfg["vocab"]
        assert not torch.equal(last(other), base), at


@pytest.mark.parametrize("batch", [2, 5, 17, 33, 70])
def test_decode_of_larger_batches(batch):
    """Batch sizes that take other product kernels (up to 4, up to 32, more rows)."""
    for dt in DT:
        cfg, w, m = make("plain", dt)
        seqs = [P.tokens(cfg, 9, seed=100 + b) for b in range(batch)]
        cache = m.new_cache(batch, 16)
        slots = cache.allocate(batch)
        m.prefill(torch.tensor([s[:6] for s in seqs], device="cuda"), [6] * batch, cache, slots)
        for t in range(6, 9):
            logits = m.decode(torch.tensor([s[t] for s in seqs], device="cuda"), cache, slots)
        some = [0, 1, batch // 3, batch // 2, batch - 2, batch - 1]
        compare(logits[some], torch.stack([reference("plain", seqs[b])[0][-1] for b in some]), dt)


def test_decode_with_the_widths_of_the_straight_line_products():
    """One sequence, bf16: widths whose matrix-vector products run without loops, with bias, squared ReLU and cap."""
    cfg = P.config([P.attention(4, 2, 16, 32, mlp=P.dense(6144)), P.hgrn2(2, 16, 16, mlp=P.dense(4096))], width=2048, vocab=64, cap=4.0)
    cfg_, w, m = make(cfg, torch.bfloat16)
    ids = P.tokens(cfg, 12)
    compare(run(m, ids, [6] + [1] * 6), O.forward(w, cfg, ids), torch.bfloat16)


@pytest.mark.parametrize("batch", [6, 16, 17, 32])
def test_decode_streams_wide_products(batch):
    """bf16 batches whose products run in each of the weight-streaming forms: wide and narrow, long and short rows, odd ends."""
    cfg = P.config([P.attention(2, 1, 16, 32, mlp=P.dense(8203)), P.hgrn2(2, 8, 16)], width=61, vocab=8301, cap=5.0)
    cfg, w, m = make(cfg, torch.bfloat16)
    seqs = [P.tokens(cfg, 6, seed=b) for b in range(batch)]
    cache = m.new_cache(batch, 8)
    slots = cache.allocate(batch)
    m.prefill(torch.tensor([s[:4] for s in seqs], device="cuda"), [4] * batch, cache, slots)
    for t in range(4, 6):
        logits = m.decode(torch.tensor([s[t] for s in seqs], device="cuda"), cache, slots)
    some = [0, 5, batch - 1]
    compare(logits[some], torch.stack([O.forward(w, cfg, seqs[b])[-1] for b in some]), torch.bfloat16)


# ---- the parts in other arrangements --------------------------------------------------------------
@pytest.mark.parametrize("dt", DT)
def test_parts_fit_other_layers(dt):
    """Gated linear and windowed latent attention in parallel layers, latents with a query latent, gates per column and per head
    with and without windows, differential attention without temperature behind norms on outputs only, plain feed-forwards with
    another activation, uncapped logits: against the oracle's pieces."""
    from oracle import gisitar_oracle as GO
    from oracle import padulorn_oracle as PO
    from vyomai_amd.layers.differential_attention import DifferentialAttention
    from vyomai_amd.layers.ffn import GatedFeedForward, PlainFeedForward
    from vyomai_amd.layers.gated_linear_attention import GatedLinearAttention
    from vyomai_amd.layers.latent_attention import LatentAttention
    from vyomai_amd.models.hybrid import HybridDecoderModel, HybridLayer, ParallelLayer
    width, vocab, eps = 40, 50, 1e-5
    hg = P.hgrn2(2, 24, 16)["mixer"]
    la = P.latent(3, 16, 8, 24, 11)["mixer"]
    at = P.attention(4, 2, 16, 24, coef=0.0, every=1)["mixer"]

    def latent(q_rank, window, head_gate):
        return LatentAttention(width, 3, 16, 8, q_rank, 24, la["scale"], eps, window, head_gate)
    layers = [ParallelLayer(width, GatedLinearAttention(width, 2, 24, 16, eps), GatedFeedForward(width, 32), eps),
              ParallelLayer(width, latent(None, 11, True), GatedFeedForward(width, 24), eps),
              HybridLayer(width, latent(20, 11, False), PlainFeedForward(width, 40, "relu2"), eps, "rms", pre=False, mult=0.5),
              HybridLayer(width, latent(20, None, True), None, eps, "rms", scalar=True),
              HybridLayer(width, DifferentialAttention(width, 4, 2, 16, 24, at["scale"], at["diff"], eps), PlainFeedForward(width, 16, "relu2"), eps,
                          "rms", pre=False),
              HybridLayer(width, latent(None, None, False), GatedFeedForward(width, 16), eps, "rms", offset=1.0)]
    gated_model = HybridDecoderModel(None, width, vocab, [layers[0], layers[1], layers[3], layers[5]], eps, "rms", embed_scale=2.0)
    plain_model = HybridDecoderModel(None, width, vocab, [layers[2], layers[3], layers[4]], eps, "rms", logit_scale=0.7, softcap=2.0, scalar=True)
    for m in (gated_model, plain_model):
        m = m.to(dt).cuda().eval()
        w = {}
        with torch.no_grad():
            for i, (n, p) in enumerate(m.named_parameters()):
                t = rnd(*p.shape, seed=i) / p.shape[-1] ** 0.5 if p.dim() > 1 else 0.3 * rnd(*p.shape, seed=i) + ("norm" in n)
                if n.endswith("lower"):
                    t = t.abs().clamp(max=0.9)
                t = t.to(torch.bfloat16).double()
                p.copy_(t)
                w[n[:-7] if n.endswith(".weight") else n] = t

        def mixer(i, h):
            mod, pre = m.layers[i].mixer, f"layers.{i}.mixer."
            p = {n[len(pre):]: t for n, t in w.items() if n.startswith(pre)}
            if mod.kind == "gated":
                return O.hgrn2(h, {"q": p["query"], "f": p["forget"], "f.b": p["forget.bias"], "lower": p["lower"], "v": p["value"], "norm": p["norm"],
                                   "o": p["out"]}, hg, eps)
            if mod.kind == "differential":
                q = {"q": p["query"], "q.b": p["query.bias"], "k": p["key"], "k.b": p["key.bias"], "v": p["value"], "v.b": p["value.bias"],
                     "q.norm": p["q_norm"], "k.norm": p["k_norm"], "o": p["out"]}
                return O.attention(h, {**q, **{n: p[n] for n in ("lq1", "lk1", "lq2", "lk2")}}, at, eps)
            q = h @ p["query"].T if mod.q_rank is None else O.rms(h @ p["q_down"].T, eps) * p["q_norm"] @ p["q_up"].T
            c = O.rms(h @ p["kv_down"].T, eps) * p["kv_norm"]
            k, v, g = c @ p["k_up"].T, c @ p["v_up"].T, O.sigmoid(h @ p["gate"].T)
            heads = [O.softmax_attention(q[:, 16 * a:16 * a + 16], k[:, 16 * a:16 * a + 16], v[:, 8 * a:8 * a + 8], la["scale"], mod.window)
                     * (g[:, a:a + 1] if mod.head_gate else g[:, 8 * a:8 * a + 8]) for a in range(3)]
            return torch.cat(heads, -1) @ p["out"].T

        def feed_forward(i, h):
            p = {n: w[f"layers.{i}.mlp.{n}"] for n in ("gate", "up", "down") if f"layers.{i}.mlp.{n}" in w}
            return GO.gated_mlp(h, p) if "gate" in p else O.mlp(h, p)

        ids = torch.randint(0, vocab, (70,), generator=torch.Generator().manual_seed(1)).tolist()
        x = m.embed_scale * w["word_embeddings"][ids]
        for i, l in enumerate(m.layers):
            def norm(t, name):
                return PO.rms_norm(t, w[f"layers.{i}.{name}"] + (1.0 if getattr(l, name).offset else 0.0), eps)
            if l.form == "parallel":
                h = norm(x, "norm1")
                x = x + mixer(i, h) + feed_forward(i, h)
            else:
                x = x + l.mult * norm(mixer(i, norm(x, "norm1") if l.pre else x), "norm1b")
                if l.mlp is not None:
                    x = x + l.mult * norm(feed_forward(i, norm(x, "norm2") if l.pre else x), "norm2b")
        want = m.logit_scale * PO.rms_norm(x, w["final_norm"], eps) @ w["head"].T
        if m.softcap is not None:
            want = O.softcap(want, m.softcap)
        for cuts in ([70], [1] * 70, [2, 1, 30, 1, 36]):
            compare(run(m, ids, cuts), want, dt)


# ---- entry points ---------------------------------------------------------------------------------
@pytest.mark.parametrize("name", list(P.CONFIGS))
def test_greedy_generation(name):
    cfg, w, m = make(name, torch.float32)
    prompts = [P.tokens(cfg, n, seed=n) for n in (5, 1, 12)]
    L, new = 12, 8
    ids = torch.tensor([p + [0] * (L - len(p)) for p in prompts], device="cuda")
    mask = torch.tensor([[1] * len(p) + [0] * (L - len(p)) for p in prompts], device="cuda")
    want = [O.greedy(w, cfg, p, new) for p in prompts]
    for kw in ({}, {"use_static_cache": True}, {"use_cache": False}):
        out = m.generate(ids, mask, max_len=new, **kw).cpu()
        assert out.shape == (3, L + new)
        for b, p in enumerate(prompts):
            n = len(p) + new
            assert out[b, :n].tolist() == want[b] and not out[b, n:].any(), kw


def test_generation_stops_and_samples():
    from vyomai_amd import NucleusProcessor, TopKProcessor, generate
    cfg, w, m = make("plain", torch.float32)
    prompt = P.tokens(cfg, 6)
    ids = torch.tensor([prompt], device="cuda")
    want = O.greedy(w, cfg, prompt, 8)
    m.config.eos_token_id = want[8]                        # the third new token (or an earlier equal one)
    end = want.index(want[8], 6)
    m.config.pad_token_id = 96
    out = m.generate(ids, max_len=8).cpu()[0].tolist()
    assert out[:end + 1] == want[:end + 1] and out[end + 1:] == [96] * (14 - end - 1)
    m.config.eos_token_id = m.config.pad_token_id = None
    assert m.generate(ids, max_len=8, processor=TopKProcessor(1.0, 1)).cpu()[0].tolist() == want
    out = m.generate(ids, max_len=8, processor=NucleusProcessor(1.0, 0.9))
    assert out.shape == (1, 14) and int(out.max()) < cfg["vocab"]
    assert generate(m, ids, max_new_tokens=8).cpu()[0].tolist() == want
    assert generate(m, ids, max_new_tokens=8, use_cache=True).cpu()[0].tolist() == want


def test_bf16_generation_follows_its_own_logits():
    cfg, _, m = make("wide", torch.bfloat16)
    prompt = P.tokens(cfg, 20)
    out = m.generate(torch.tensor([prompt], device="cuda"), max_len=12).cpu()[0].tolist()
    logits = run(m, out, [20] + [1] * 12)
    assert out[20:] == logits[19:-1].float().argmax(-1).tolist()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_replay(dtype, tmp_path):
    cfg = P.CONFIGS["odd"]
    w = P.weights(cfg)
    P.write_folder(tmp_path, cfg, w)
    a, b = P.tokens(cfg, 60, seed=1), P.tokens(cfg, 12, seed=2)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:50], "want": [0, 49]}, {"id": "b", "tokens": b[:10], "want": [9]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[50:51], "want": []}, {"id": "b", "tokens": b[10:11], "want": [0]}], "end": ["b"]},
             {"step": 2, "entries": [{"id": "a", "tokens": a[51:52], "want": []}], "end": []},
             {"step": 3, "entries": [{"id": "a", "tokens": a[52:], "want": [7]}], "end": ["a"]},
             {"step": 4, "entries": [{"id": "b", "tokens": b[:1], "want": [0]}], "end": ["b"]}]
    r = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", str(tmp_path), "--dtype", dtype,
                        "--out", str(tmp_path), "--max-tokens", "96"], input="\n".join(json.dumps(s) for s in steps) + "\n",
                       capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [l for l in r.stdout.splitlines() if l.startswith("done")] == [f"done {i}" for i in range(5)]
    fa, fb = O.forward(w, cfg, a), O.forward(w, cfg, b)
    want = {0: torch.stack([fa[0], fa[49], fb[9]]), 1: fb[10:11], 3: fa[59:60], 4: fb[:1]}
    assert {int(f.stem) for f in tmp_path.glob("*.f32")} == set(want)
    for i, t in want.items():
        got = torch.frombuffer(bytearray((tmp_path / f"{i}.f32").read_bytes()), dtype=torch.float32).view(-1, cfg["vocab"])
        assert got.shape == t.shape
        compare(got, t, torch.float32 if dtype == "float32" else torch.bfloat16)
