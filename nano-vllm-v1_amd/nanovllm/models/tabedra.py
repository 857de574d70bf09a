"""Tabedra: a decoder-only stack over a residual stream that is kept in several fp32 copies (hyper-connections), with windowed softmax
attention whose scores carry a learned distance bias and mixture-of-experts feed-forwards of ungated squared-ReLU experts.

    e = embed[token] + bigram[(previous token * mul_prev + token * mul_cur) mod buckets] + pos[position]       (first token: the last bigram row)
    x_1 .. x_S = e
    for every layer, for its mixer (q = 1) and then its feed-forward (q = 2; layers without one skip it):
        u = sum_s in_q[s] x_s;   y = sublayer(norm_q(u));   x_t <- sum_s mix_q[s, t] x_s + out_q[t] y          (layers.hyper.HyperConnection)
    logits = head final_norm(sum_s x_s)
(all norms are affine layer norms)

Mixer `attention` (layers.attention.WindowedBiasAttention): q, k, v without biases and without rotation; a short causal convolution over time per
channel right after each projection; q and k divided by their root mean square per head; score = scale q.k + rel[bucket(distance), head]; a
sliding window; the concatenated heads times sigmoid(W_g h) element by element.  A layer with `kv_from: j` has queries only and reads the
keys and values that layer j cached.
Feed-forward: layers.moe.SparseMoE with score="softmax_all": a correction that steers the choice only, the chosen scores divided by their
sum; ungated experts down(relu(up x)^2), a shared one of the same form for every token.

A sequence's state beside its pages: the last conv - 1 projected rows of every attention layer and the last token id (for the bigram).

32-bit whatever the activation type: positions, every norm, attention scores, their bias and weights, router logits and scores, the streams,
their coefficients and sums, the convolutions' sums and the root mean squares.  Projections run in the model's dtype (bf16, or fp32 for a
model served in full precision).

config.json keys: architecture, vocab, width, max_positions, streams, norm.eps, embedding {bigram {buckets, mul_prev, mul_cur}}, layers[] of
{type: attention, mixer {heads, kv_heads, dim, vdim, conv, scale, bias_max, mask {size} | null, kv_from}, mlp {kind: moe, expert {ff},
router {experts, top}, shared {ff} | null} | null}; the rows of a distance-bias table come from the checkpoint's shape.  Tensors: embed, bigram,
pos, head, final.norm(.b), l<i>.norm1|norm2(.b), l<i>.hc1|hc2.in|out|mix, l<i>.mix.q|k|v(.conv)|rel|g|o, l<i>.mlp.e<n>.up|down,
l<i>.mlp.router|correction, l<i>.mlp.shared.up|down.
"""
from __future__ import annotations

import re
import zlib

import torch
from torch import nn

from .. import ops
from ..layers.attention import WindowedBiasAttention
from ..layers.hyper import HyperConnection
from ..layers.layernorm import StreamNorm
from ..layers.linear import MergedLinear
from ..layers.moe import SparseMoE
from ..layers.state import LastToken
from ..utils.context import get_context
from .lamutar import _get


class TabedraAttention(nn.Module):
    def __init__(self, width: int, m, eps: float, bias_rows: int, source: "TabedraAttention | None"):
        super().__init__()
        h, d = int(_get(m, "heads")), int(_get(m, "dim"))
        g, dv = int(_get(m, "kv_heads", h)), int(_get(m, "vdim", d))
        mask = _get(m, "mask")
        self.attn = WindowedBiasAttention(h, g, d, dv, float(_get(m, "scale", d ** -0.5)), None, window=int(_get(mask, "size", 0) or 0) if mask else 0,
                                          distance_bias=(bias_rows, int(_get(m, "bias_max"))), conv=int(_get(m, "conv", 0) or 0), unit_qk=eps, gated="element",
                                          kv_source=None if source is None else source.attn)
        names = ["q", "g"] if source is not None else ["q", "k", "v", "g"]
        self.proj = MergedLinear(width, self.attn.projection_sizes(), names)
        self.o = MergedLinear(h * dv, [width])

    def forward(self, x: torch.Tensor, positions: torch.Tensor) -> dict:
        return dict(a=self.o(self.attn(self.proj(x), positions)))


class TabedraLayer(nn.Module):
    def __init__(self, width: int, spec, eps: float, streams: int, bias_rows: int, source: TabedraAttention | None):
        super().__init__()
        kind, mixer, mlp = _get(spec, "type"), _get(spec, "mixer"), _get(spec, "mlp")
        if kind != "attention":
            raise ValueError(f"unknown mixer type {kind!r}")
        self.mixer = TabedraAttention(width, mixer, eps, bias_rows, source)
        self.norm1, self.hc1 = StreamNorm(width, eps, "layer"), HyperConnection(streams)
        self.mlp = None
        if mlp:
            if _get(mlp, "kind", "moe") != "moe":
                raise ValueError(f"unknown feed-forward kind {_get(mlp, 'kind')!r}")
            router, shared = _get(mlp, "router"), _get(mlp, "shared")
            self.mlp = SparseMoE(width, int(_get(_get(mlp, "expert"), "ff")), int(_get(router, "experts")), int(_get(router, "top")),
                                 shared_ff=int(_get(shared, "ff")) if shared else None, act="relu2", router_bias=False, score="softmax_all", correction=True,
                                 renormalize=True, gated=False)
            self.norm2, self.hc2 = StreamNorm(width, eps, "layer"), HyperConnection(streams)


class TabedraForCausalLM(nn.Module):
    requires_cache = True            # attention reads its keys from the paged cache in every step (no packed mode)
    has_recurrent_state = True       # sequences hold a state slot; cached pages cannot stand in for a prefix
    supported_dtypes = (torch.bfloat16, torch.float32)
    DEFAULT_BIAS_ROWS = 32

    def __init__(self, config) -> None:
        super().__init__()
        self.config = config
        width, vocab = int(config.width), int(config.vocab)
        eps = float(_get(config.norm, "eps", 1e-6))
        self.width, self.vocab, self.streams = width, vocab, int(getattr(config, "streams", 1) or 1)
        bigram = _get(getattr(config, "embedding", None) or {}, "bigram")
        self.embed = MergedLinear(width, [vocab])            # [vocab, width]: a table, stored like a projection
        self.pos = nn.Parameter(torch.zeros(int(config.max_positions), width), requires_grad=False)
        if bigram:
            self.bigram = nn.Parameter(torch.zeros(int(_get(bigram, "buckets")) + 1, width), requires_grad=False)
            self.bigram_factors = int(_get(bigram, "mul_prev")), int(_get(bigram, "mul_cur"))
            self.last_token = LastToken()
        else:
            self.register_parameter("bigram", None)
        rows = getattr(config, "bias_rows", None) or {}
        self.layers = nn.ModuleList()
        for i, spec in enumerate(config.layers):
            j = _get(_get(spec, "mixer"), "kv_from")
            if j is not None and not 0 <= int(j) < i:
                raise ValueError(f"layer {i} reads the keys of layer {j}, which does not run before it")
            self.layers.append(TabedraLayer(width, spec, eps, self.streams, rows.get(i, self.DEFAULT_BIAS_ROWS), None if j is None else self.layers[int(j)].mixer))
        self.final_norm = StreamNorm(width, eps, "layer")
        self.head = MergedLinear(width, [vocab])
        self.collect = None          # a list: receives the sum of the streams after every layer (debugging, tests)

    # ------------------------------------------------------------------ checkpoint names
    def weight_target(self, name: str):
        """(parameter name, shard id | None) of a checkpoint tensor; (None, None) for one that is stored and not used."""
        top = {"embed": "embed.weight", "head": "head.weight", "pos": "pos", "bigram": "bigram", "final.norm": "final_norm.weight", "final.norm.b": "final_norm.bias"}
        if name in top:
            return top[name], None
        m = re.fullmatch(r"l(\d+)\.(.+)", name)
        if not m or int(m.group(1)) >= len(self.layers):
            raise KeyError(f"checkpoint tensor {name!r} matches no parameter of the model")
        i, rest = int(m.group(1)), m.group(2)
        p, layer = f"layers.{i}.", self.layers[i]
        around = re.fullmatch(r"(?:norm([12])(\.b)?|hc([12])\.(in|out|mix))", rest)
        if around:
            q = around.group(1) or around.group(3)
            if q == "2" and layer.mlp is None:
                return None, None
            if around.group(1):
                return p + f"norm{q}." + ("bias" if around.group(2) else "weight"), None
            return p + f"hc{q}." + {"in": "in_weights", "out": "out_weights", "mix": "mix"}[around.group(4)], None
        if rest.startswith("mix."):
            leaf, pm, mixer = rest[4:], p + "mixer.", layer.mixer
            if leaf in ("o", "rel"):
                return pm + {"o": "o.weight", "rel": "attn.bias"}[leaf], None
            if leaf in mixer.proj.shard_ids:
                return pm + "proj.weight", leaf
            conv = mixer.attn.conv_weight
            if leaf.endswith(".conv") and conv is not None and leaf[:-5] in conv.shard_ids:
                return pm + "attn.conv_weight", leaf[:-5]
        elif rest.startswith("mlp.") and layer.mlp is not None:
            leaf, pm = rest[4:], p + "mlp."
            direct = {"router": "router.weight", "correction": "correction"}
            if layer.mlp.shared is not None:
                direct.update({"shared.up": "shared.up.weight", "shared.down": "shared.down.weight"})
            if leaf in direct:
                return pm + direct[leaf], None
            e = re.fullmatch(r"e(\d+)\.(up|down)", leaf)
            if e and int(e.group(1)) < layer.mlp.experts:
                n = int(e.group(1))
                return (pm + "down", n) if e.group(2) == "down" else (pm + "gate_up", (n, "up"))
        raise KeyError(f"checkpoint tensor {name!r} matches no parameter of the model")

    @staticmethod
    def adapt_config(config, shapes: dict) -> None:
        """Sizes that only the checkpoint's tensor shapes give: the rows of each layer's distance-bias table (`shapes`: tensor name ->
        shape; empty without a checkpoint, then a default is used)."""
        config.bias_rows = {int(m.group(1)): int(shape[0]) for m, shape in ((re.fullmatch(r"l(\d+)\.mix\.rel", name), shape) for name, shape in shapes.items()) if m}
        if not hasattr(config, "max_positions"):
            config.max_positions = int(shapes["pos"][0]) if "pos" in shapes else 4096

    @staticmethod
    def synthetic_tensors(config, seed: int = 0, std: float = 0.02, device="cuda", dtype=torch.bfloat16):
        """Random weights in checkpoint naming (for benchmarks and smoke runs without a checkpoint)."""
        width, vocab, streams = int(config.width), int(config.vocab), int(getattr(config, "streams", 1) or 1)
        rows = getattr(config, "bias_rows", None) or {}

        def mat(name, *shape, scale=std, shift=0.0):
            g = torch.Generator(device=device)
            g.manual_seed((zlib.crc32(name.encode()) ^ (seed * 0x9E3779B1)) & 0x7FFFFFFF)
            return name, (torch.randn(tuple(shape), generator=g, device=device, dtype=torch.float32) * scale + shift).to(dtype)

        yield mat("embed", vocab, width, scale=1.0)
        yield mat("pos", int(config.max_positions), width, scale=0.1)
        bigram = _get(getattr(config, "embedding", None) or {}, "bigram")
        if bigram:
            yield mat("bigram", int(_get(bigram, "buckets")) + 1, width, scale=0.5)
        yield mat("head", vocab, width)
        yield mat("final.norm", width, scale=0.1, shift=1.0)
        yield mat("final.norm.b", width, scale=0.1)
        for i, spec in enumerate(config.layers):
            p, m, mlp = f"l{i}.", _get(spec, "mixer"), _get(spec, "mlp")
            for q in (1, 2) if mlp else (1,):
                yield mat(p + f"norm{q}", width, scale=0.1, shift=1.0)
                yield mat(p + f"norm{q}.b", width, scale=0.1)
                yield mat(p + f"hc{q}.in", streams, scale=0.1, shift=1.0 / streams)
                yield mat(p + f"hc{q}.out", streams, scale=0.1, shift=1.0)
                name, noise = mat(p + f"hc{q}.mix", streams, streams, scale=0.1)
                yield name, noise + torch.eye(streams, device=device, dtype=dtype)
            h, d = int(_get(m, "heads")), int(_get(m, "dim"))
            g, dv, conv = int(_get(m, "kv_heads", h)), int(_get(m, "vdim", d)), int(_get(m, "conv", 0) or 0)
            own = _get(m, "kv_from") is None
            for leaf, n in [("q", h * d)] + ([("k", g * d), ("v", g * dv)] if own else []):
                yield mat(p + "mix." + leaf, n, width)
                if conv:
                    yield mat(p + f"mix.{leaf}.conv", n, conv, scale=0.4)
            yield mat(p + "mix.rel", rows.get(i, TabedraForCausalLM.DEFAULT_BIAS_ROWS), h, scale=0.5)
            yield mat(p + "mix.g", h * dv, width)
            yield mat(p + "mix.o", width, h * dv)
            if not mlp:
                continue
            ff, router, shared = int(_get(_get(mlp, "expert"), "ff")), _get(mlp, "router"), _get(mlp, "shared")
            for e in range(int(_get(router, "experts"))):
                yield mat(f"{p}mlp.e{e}.up", ff, width)
                yield mat(f"{p}mlp.e{e}.down", width, ff)
            yield mat(p + "mlp.router", int(_get(router, "experts")), width)
            yield mat(p + "mlp.correction", int(_get(router, "experts")), scale=0.02)
            if shared:
                yield mat(p + "mlp.shared.up", int(_get(shared, "ff")), width)
                yield mat(p + "mlp.shared.down", width, int(_get(shared, "ff")))

    # ------------------------------------------------------------------ forward
    def forward(self, input_ids: torch.Tensor, positions: torch.Tensor) -> torch.Tensor:
        """The fp32 streams [T, S, width] after the last layer (their sum and the final norm are formed of the rows that are projected)."""
        ctx = get_context()
        pairs = {} if self.bigram is None else dict(bigram=self.bigram.data, mul_prev=self.bigram_factors[0], mul_cur=self.bigram_factors[1], last_tokens=self.last_token.ids(),
                                                    slots=ctx.state_slots, cu_seqlens_q=ctx.cu_seqlens_q, context_lens=ctx.context_lens)
        x = ops.embedding_bigram_stream(input_ids, positions, self.embed.weight.data, self.streams, self.pos.data, **pairs)
        h = self.layers[0].hc1.open(x, self.layers[0].norm1)
        for layer, after in zip(self.layers, list(self.layers)[1:] + [None]):
            opening = None if after is None else (after.hc1, after.norm1)
            terms = layer.mixer(h, positions)
            if layer.mlp is not None:
                h = layer.hc1.close(x, terms, (layer.hc2, layer.norm2))
                h = layer.hc2.close(x, layer.mlp.terms(h), opening)
            else:
                h = layer.hc1.close(x, terms, opening)
            if self.collect is not None:
                self.collect.append(x.sum(1))
        return x

    def gather_rows(self, hidden: torch.Tensor, rows: torch.Tensor) -> torch.Tensor:
        return ops.gather_rows_f32(hidden.view(hidden.shape[0], -1), rows)

    def compute_logits_rows(self, rows: torch.Tensor) -> torch.Tensor:
        """fp32 logits [R, vocab] of selected rows of the streams: their sum, final norm, head."""
        return self.head(ops.hyper_norm(rows.reshape(-1, self.streams, self.width), **self.final_norm.spec()), out_f32=True)

    def compute_logits(self, hidden: torch.Tensor) -> torch.Tensor:
        return self.compute_logits_rows(hidden)
