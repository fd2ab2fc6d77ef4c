"""Decoders that mix layer kinds over an fp32 residual stream: every layer is one mixer (latent attention, lightning attention,
windowed attention, ...) and an optional feed-forward (gated, plain, or a mixture of experts), in one of two forms:

    HybridLayer    x <- x + m norm1b(mixer(norm1(x))) ;  x <- x + m norm2b(ff(norm2(x)))    (without norm1 / norm2: of x itself)
    ParallelLayer  x <- x + (mixer(h) + ff(h)),  h = norm1(x)

A design built from this file supplies its layers and its parameter names (models/gisitar.py, rivudra.py, padulorn.py,
biruvik.py); embedding, residual stream, slot cache, prefill, the native single-token step and generation are here.  Inference only.
"""
from __future__ import annotations

import functools
from typing import List, Optional, Sequence

import torch
import torch.nn as nn

from .. import ops
from .._lib import VyomHipError
from ..layers.kv_cache import SlotCache
from ..layers.norms import WeightNorm
from ..layers.packing import Packed, norm_vec, pad2
from ..ops import up8
from .decoder import CLMOutput


class HybridLayer(nn.Module):
    """One mixer and (mlp may be None) one feed-forward behind it, with norms ahead of them (pre) and on their outputs, which
    join the residual stream times `mult`."""
    form = "sandwich"

    def __init__(self, width: int, mixer: nn.Module, mlp: Optional[nn.Module], eps: float, norm: str = "layer",
                 offset: float = 0.0, pre: bool = True, mult: float = 1.0, scalar: bool = False) -> None:
        """scalar: the norms' weights are one number each."""
        super().__init__()
        self.mixer, self.mlp, self.width, self.pre, self.mult = mixer, mlp, width, pre, float(mult)
        for n in self._norms():
            setattr(self, n, WeightNorm(width, eps, norm, offset, scalar))

    def _norms(self) -> List[str]:
        names = ["norm1", "norm1b"] + (["norm2", "norm2b"] if self.mlp is not None else [])
        return [n for n in names if self.pre or n.endswith("b")]

    def packed(self) -> Packed:
        def build(p: Packed) -> None:
            p.norm1 = p.norm2 = ops.PLAIN
            for n in self._norms():
                setattr(p, n, norm_vec(getattr(self, n), up8(self.width), self.mult if n.endswith("b") else 1.0))
        return Packed.of(self, [getattr(self, n).weight for n in self._norms()], build)

    def run(self, norm, h: torch.Tensor, B: int, L: int, batch, layer: int, nxt: Optional[torch.Tensor]) -> Optional[torch.Tensor]:
        """h = norm1(x) (or x) of the new tokens; norm(y=, post=, pre=, routed=) advances the residual stream x by a sublayer and
        returns its next norm.  nxt: the norm of what follows this layer."""
        p = self.packed()
        y = self.mixer(h, B, L, batch, layer)
        if self.mlp is None:
            return norm(y=y, post=p.norm1b, pre=nxt)
        h = norm(y=y, post=p.norm1b, pre=p.norm2)
        routed = self.mlp.routed(h, L, batch.count)
        return norm(y=self.mlp.dense(h) if self.mlp.dense is not None else None, routed=routed, post=p.norm2b, pre=nxt)


class ParallelLayer(nn.Module):
    """One norm whose output both the mixer and (mlp may be None) the feed-forward read.  The projections of the mixer and of
    the feed-forward's dense part are ONE product of h, and their output products are one as well."""
    form = "parallel"

    def __init__(self, width: int, mixer: nn.Module, mlp: Optional[nn.Module], eps: float, norm: str = "rms",
                 offset: float = 0.0) -> None:
        super().__init__()
        self.mixer, self.mlp, self.width = mixer, mlp, width
        self.norm1 = WeightNorm(width, eps, norm, offset)

    @property
    def dense(self):
        return self.mlp.dense if self.mlp is not None else None

    def packed(self) -> Packed:
        params = [self.norm1.weight, *self.mixer.parameters(), *(self.dense.parameters() if self.dense is not None else [])]

        def build(p: Packed) -> None:
            p.norm1 = norm_vec(self.norm1, up8(self.width))
            if getattr(self.mixer, "query", None) is not None and self.mixer.query.bias is not None:
                raise ValueError("a mixer with biases does not share its products (no parallel layers)")
            p.w_in, p.w_o = self.mixer.matrices()
            p.n_mix, p.n_heads = p.w_in.shape[0], p.w_o.shape[1]
            if self.dense is not None:
                gate_up, down = self.dense.matrices()
                p.w_in, p.w_o = torch.cat([p.w_in, gate_up]), torch.cat([p.w_o, down], 1)
            p.w_in, p.w_o = p.w_in.contiguous(), p.w_o.contiguous()
        return Packed.of(self, params, build)

    def run(self, norm, h: torch.Tensor, B: int, L: int, batch, layer: int, nxt: Optional[torch.Tensor]) -> Optional[torch.Tensor]:
        p = self.packed()
        rows = ops.linear(h, p.w_in)
        both = torch.empty((B * L, p.w_o.shape[1]), dtype=h.dtype, device=h.device)
        self.mixer.mix(rows[:, : p.n_mix], B, L, batch, layer, out=both[:, : p.n_heads])
        if self.dense is not None:
            self.dense.activation(rows[:, p.n_mix:], out=both[:, p.n_heads:])
        routed = self.mlp.routed(h, L, batch.count) if self.mlp is not None else None
        return norm(y=ops.linear(both, p.w_o), routed=routed, pre=nxt)


class HybridDecoderModel(nn.Module):
    """`layers` of HybridLayer / ParallelLayer between a (scaled) embedding and a norm + vocabulary projection (softcap: logits
    become softcap tanh(logits / softcap); scalar: the norm's weight is one number)."""

    def __init__(self, config, width: int, vocab: int, layers: Sequence[nn.Module], eps: float, norm: str = "layer",
                 offset: float = 0.0, embed_scale: float = 1.0, logit_scale: float = 1.0, softcap: Optional[float] = None,
                 scalar: bool = False) -> None:
        super().__init__()
        self.config, self.width, self.vocab, self.eps, self.rms = config, width, vocab, float(eps), norm == "rms"
        self.embed_scale, self.logit_scale = float(embed_scale), float(logit_scale)
        self.softcap = float(softcap) if softcap is not None else None
        if softcap is not None and not softcap > 0:
            raise ValueError(f"logits capped at {softcap}")
        self.word_embeddings = nn.Embedding(vocab, width)
        self.layers = nn.ModuleList(layers)
        self.final_norm = WeightNorm(width, eps, norm, offset, scalar)
        self.head = nn.Linear(width, vocab, bias=False)
        self._own_cache: Optional[SlotCache] = None
        self.requires_grad_(False)

    # ---- kernel-side tensors ----------------------------------------------------------------
    @property
    def dtype(self) -> torch.dtype:
        return self.word_embeddings.weight.dtype

    @property
    def device(self) -> torch.device:
        return self.word_embeddings.weight.device

    def packed(self) -> Packed:
        def build(p: Packed) -> None:
            dp = up8(self.width)
            p.embed = pad2(self.word_embeddings.weight, self.vocab, dp).contiguous()
            p.head = pad2(self.head.weight, self.vocab, dp).contiguous()
            p.final_norm = norm_vec(self.final_norm, dp, self.logit_scale)   # (the head is linear)
        return Packed.of(self, [self.word_embeddings.weight, self.head.weight, self.final_norm.weight], build)

    # ---- cache ------------------------------------------------------------------------------
    def new_cache(self, slots: int = 1, capacity: int = 64) -> SlotCache:
        """Memory for `slots` sequences of `capacity` tokens (both grow)."""
        return SlotCache([l.mixer.cache_spec() for l in self.layers], self.dtype, self.device, slots, capacity)

    # ---- forward ----------------------------------------------------------------------------
    def prefill(self, tokens: torch.Tensor, counts: Sequence[int], cache: SlotCache, slots: Sequence[int],
                layers_out: Optional[list] = None) -> torch.Tensor:
        """tokens (B, L), the first counts[b] of row b real: runs them behind what slots[b] holds -> residual stream
        (B, L, padded width) fp32.  Logits of chosen rows: ``logits(rows)``."""
        if not tokens.is_cuda:
            raise VyomHipError("vyomai_amd ops run on MI355X only: got CPU token ids (no CPU fallback exists; move the "
                               "model and its inputs to 'cuda')")
        B, L = tokens.shape
        batch = cache.reserve(list(slots), list(counts))
        p = self.packed()
        dp = up8(self.width)
        x = torch.empty((B * L, dp), dtype=torch.float32, device=tokens.device)
        norms = [l.packed() for l in self.layers]
        norm = functools.partial(ops.residual_norm, x, self.width, eps=self.eps, rms=self.rms)
        h = norm(table=p.embed, ids=tokens.reshape(-1).contiguous(), table_scale=self.embed_scale, pre=norms[0].norm1)
        for i, layer in enumerate(self.layers):
            # (the last layer's stream is normed row by row in logits(): only the rows asked for)
            h = layer.run(norm, h, B, L, batch, i, norms[i + 1].norm1 if i + 1 < len(self.layers) else None)
            if layers_out is not None:
                layers_out.append(x.view(B, L, dp)[..., : self.width].clone())
        cache.advance(list(slots), list(counts))
        return x.view(B, L, dp)

    def logits(self, rows: torch.Tensor) -> torch.Tensor:
        """Residual rows (M, padded width) -> logits (M, vocab)."""
        p = self.packed()
        rows = rows if rows.stride(1) == 1 else rows.contiguous()
        h = ops.residual_norm(rows, self.width, pre=p.final_norm, eps=self.eps, rms=self.rms, dtype=self.dtype)
        return ops.linear(h, p.head) if self.softcap is None else ops.linear_softcap(h, p.head, self.softcap)

    def decode(self, ids: torch.Tensor, cache: SlotCache, slots: Sequence[int]) -> torch.Tensor:
        """One more token (ids (B,) int64 on the device) for each sequence: ONE native call -> logits (B, vocab)."""
        from ..decode_plan import HybridDecodePlan
        slots = list(slots)
        batch = cache.reserve(slots, [1] * len(slots))
        # plans live with the cache whose buffers they point at; a model that was given other weights is another owner
        key = id(self), self.word_embeddings.weight.data_ptr(), self.head.weight.data_ptr(), len(slots)
        plan = cache.plans.get(key)
        if plan is None or not plan.valid(cache):
            if len(cache.plans) > 8:
                cache.plans.clear()
            plan = cache.plans[key] = HybridDecodePlan(self, cache, len(slots))
        out = plan.step(ids, batch)
        cache.advance(slots, [1] * len(slots), on_device=False)
        return out

    @staticmethod
    def _counts(input_ids: torch.Tensor, attention_mask: Optional[torch.Tensor]) -> List[int]:
        B, L = input_ids.shape
        if attention_mask is None:
            return [L] * B
        keep = attention_mask[:, -L:].to(torch.int64).cpu()
        counts = keep.sum(1)
        if not bool((keep == (torch.arange(L)[None] < counts[:, None])).all()) or int(counts.min()) < 1:
            raise ValueError("padding must follow the tokens of a sequence (and every sequence needs a token): the layers' "
                             "states run over the tokens in order")
        return counts.tolist()

    @torch.no_grad()
    def forward(self, input_ids: torch.Tensor, attention_mask: Optional[torch.Tensor] = None, use_cache: bool = False,
                kv_cache: Optional[SlotCache] = None, start_pos: int = 0, slots: Optional[Sequence[int]] = None) -> CLMOutput:
        """Logits of every position.  use_cache without kv_cache: the model's own cache, emptied by start_pos = 0 (what
        generation_utils.generate drives).  slots: the cache slots of the rows (default 0 .. B-1 of a cache made here)."""
        B, L = input_ids.shape
        counts = self._counts(input_ids, attention_mask)
        cache = kv_cache
        if cache is None:
            if use_cache and start_pos > 0:
                cache = self._own_cache
                if cache is None:
                    raise ValueError("start_pos > 0 without a cached prefix")
            else:
                cache = self.new_cache(B, L if not use_cache else max(64, 2 * L))
                slots = cache.allocate(B)
                self._own_cache = cache if use_cache else None
        if slots is None:
            slots = list(range(B))
        hidden = self.prefill(input_ids, counts, cache, slots)
        logits = self.logits(hidden.view(B * L, -1)).view(B, L, -1)
        return CLMOutput(hidden_state=hidden[..., : self.width], logits=logits, kv_cache=cache if use_cache else None)

    # ---- generation -------------------------------------------------------------------------
    @torch.no_grad()
    def generate(self, input_ids: torch.Tensor, attention_mask: Optional[torch.Tensor] = None, max_len: int = 5,
                 temperature: float = 1.0, use_cache: bool = True, do_sample: bool = False,
                 use_static_cache: bool = False, processor=None) -> torch.Tensor:
        """Batched generation: prompts of unequal length padded behind (attention_mask tells), max_len new tokens each.
        Returns (B, prompt + max_len): row b holds its prompt, then its tokens, then padding; a row stops at an
        end-of-sequence id of the config.  processor: one of logits_processors (top-k, nucleus, ...); do_sample draws from
        softmax(logits / temperature); otherwise greedy.  use_static_cache: size the cache for the whole run at once."""
        from ..logits_processors import MultinomialProcessor
        dev = input_ids.device
        B, P = input_ids.shape
        counts = self._counts(input_ids, attention_mask)
        pad = getattr(self.config, "pad_token_id", None) or 0
        eos = getattr(self.config, "eos_token_id", None)
        eos = [] if eos is None else list(eos) if isinstance(eos, (list, tuple)) else [eos]
        eos_ids = torch.tensor(eos or [-1], dtype=torch.long, device=dev)
        if do_sample and processor is None:
            processor = MultinomialProcessor(temperature)
        new = torch.full((B, max_len), pad, dtype=torch.long, device=dev)
        done = torch.zeros(B, dtype=torch.bool, device=dev)
        left = torch.zeros(max_len, dtype=torch.int32, device=dev)
        out = torch.full((B, P + max_len), pad, dtype=torch.long, device=dev)
        for b, n in enumerate(counts):
            out[b, :n] = input_ids[b, :n]

        def first_logits(cache, slots, ids, n):
            hidden = self.prefill(ids, n, cache, slots)
            rows = torch.tensor([b * ids.shape[1] + c - 1 for b, c in enumerate(n)], device=dev)
            return self.logits(hidden.view(-1, hidden.shape[-1]).index_select(0, rows))

        cache = self.new_cache(B, P + max_len if use_static_cache else P)
        slots = cache.allocate(B)
        logits = first_logits(cache, slots, input_ids, counts) if max_len else None
        steps = 0
        for i in range(max_len):
            if i:
                if use_cache:
                    logits = self.decode(new[:, i - 1].contiguous(), cache, slots)
                else:
                    cache.free(slots)
                    slots = cache.allocate(B)
                    logits = first_logits(cache, slots, out[:, : P + i], [n + i for n in counts])
            if processor is None:
                ops.greedy_step_(logits, new, i, None, eos_ids, done, left[i:i + 1])
            else:
                token = processor.sample(processor(logits.float())).reshape(-1)
                new[:, i] = torch.where(done, torch.full_like(token, pad), token)
                done |= torch.isin(token, eos_ids)
                left[i] = (~done).sum()
            steps = i + 1
            if not use_cache:
                for b, n in enumerate(counts):
                    out[b, n + i] = new[b, i]
            if eos and int(left[i]) == 0:
                break
        if eos:   # (greedy rows run on behind their end while others are busy)
            hit = torch.isin(new[:, :steps], eos_ids).int().cumsum(1)
            ended = (hit - torch.isin(new[:, :steps], eos_ids).int()) > 0
            new[:, :steps] = torch.where(ended, torch.full_like(new[:, :steps], pad), new[:, :steps])
        for b, n in enumerate(counts):
            out[b, n:n + max_len] = new[b]
            out[b, n + max_len:] = pad
        return out
