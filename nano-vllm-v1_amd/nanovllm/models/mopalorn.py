"""Mopalorn: a decoder-only stack over an fp32 residual stream with an RMS norm before and after every sublayer, three kinds of softmax
attention and an ungated xIELU feed-forward.

    x = embed[token]
    for every layer:
        x = x + norm1b(mixer(norm1(x)))
        x = x + norm2b(ff(norm2(x)))                   (layers without a feed-forward skip this)
    logits = logit_scale * embed final_norm(x)         (the embedding table is the output projection too)

Mixers (sizes and constants per layer from config.json):
  latent_attention  keys and values from one cached normed latent and one cached rotated key part shared by the heads (rotary in the
                    halves layout), queries straight from the input, a sliding window, a sigmoid gate per output element
                    (layers.attention.LatentAttention)
  attention         q, k, v without biases and without rotation; a query temperature that grows with the position's logarithm, a
                    softcap on the scores, every earlier token visible
  attention_2       q, k, v without biases and without rotation; a sliding window, before it one mean key and value per block of
                    `mask.pool` positions, and a sink logit per head
                    (both layers.attention.WindowedBiasAttention)
Value mixing: of the layers that say `v_mix`, the first keeps its own values and hands them on; every later one caches
(1 - l) v + l v_first of the same token, with a learned number l.
Feed-forward: down(xielu(up x)).

32-bit whatever the activation type: positions and angles, the query temperature, attention scores, their softcap, sinks and weights, the
means' sums, every norm, the residual stream and its sums.  Projections run in the model's dtype (bf16, or fp32 for a model served in
full precision).  No layer keeps a state beside its pages, so prompts with a common prefix share pages (and the block means in them).

config.json keys: architecture, vocab, width, norm.eps, logit_scale, layers[] of {type, mixer {...}, mlp {kind: dense, ff} | null}.
latent_attention mixer: heads, dim, rot_dim, vdim, kv_rank, scale, rot {base, dims}, mask {size} | null; attention: heads, kv_heads, dim,
vdim, scale, softcap, q_temp {coef, every}, v_mix; attention_2: heads, kv_heads, dim, vdim, scale, mask {size, pool}, v_mix.
Tensors: embed, final.norm, l<i>.norm1|norm1b|norm2|norm2b, l<i>.mix.q|dkv|dkv.norm|uk|uv|g|o (latent_attention),
l<i>.mix.q|k|v|o|vmix|sink (the others), l<i>.mlp.up|down|act.
"""
from __future__ import annotations

import re
import zlib

import torch
from torch import nn

from .. import ops
from ..layers.activation import XIELU
from ..layers.attention import LatentAttention, WindowedBiasAttention
from ..layers.layernorm import StreamNorm
from ..layers.linear import MergedLinear
from ..layers.rotary_embedding import rotary_frequencies
from .lamutar import _get


class MopalornLatentAttention(nn.Module):
    def __init__(self, width: int, m, eps: float):
        super().__init__()
        h, d, dr = int(_get(m, "heads")), int(_get(m, "dim")), int(_get(m, "rot_dim", 0) or 0)
        dv, rank = int(_get(m, "vdim", d)), int(_get(m, "kv_rank"))
        rot, mask = _get(m, "rot"), _get(m, "mask")
        assert dr == 0 or int(_get(rot, "dims", dr)) == dr, "the rotated part is the whole of rot_dim"
        freq, mag = rotary_frequencies(dr, float(_get(rot, "base", 10000.0))) if dr else (None, 1.0)
        self.attn = LatentAttention(h, d, dr, dv, None, rank, float(_get(m, "scale", (d + dr) ** -0.5)), eps, freq, mag, interleaved=False, gated="element",
                                    window=int(_get(mask, "size", 0) or 0) if mask else 0)
        self.proj = MergedLinear(width, self.attn.projection_sizes(), ["q", "dkv", "g"])
        self.o = MergedLinear(h * dv, [width])

    def forward(self, x: torch.Tensor, positions: torch.Tensor, v_first) -> tuple[torch.Tensor, None]:
        return self.o(self.attn(self.proj(x), positions)), None


class MopalornAttention(nn.Module):
    """`pooled`: the variant with a window, block means before it and sinks; else the one over all earlier tokens with query temperature
    and softcap.  `mixes`: an earlier layer's values are mixed in."""

    def __init__(self, width: int, m, pooled: bool, mixes: bool):
        super().__init__()
        h, d = int(_get(m, "heads")), int(_get(m, "dim"))
        g, dv = int(_get(m, "kv_heads", h)), int(_get(m, "vdim", d))
        mask, temp = _get(m, "mask"), _get(m, "q_temp")
        special = (dict(window=int(_get(mask, "size")), pool=int(_get(mask, "pool", 0) or 0), sinks=True) if pooled else
                   dict(softcap=float(_get(m, "softcap", 0.0) or 0.0), q_temp=(float(_get(temp, "coef")), int(_get(temp, "every"))) if temp else None))
        self.sizes = [h * d, g * d, g * dv]
        self.proj = MergedLinear(width, self.sizes, ["q", "k", "v"])
        self.attn = WindowedBiasAttention(h, g, d, dv, float(_get(m, "scale", d ** -0.5)), None, mix_values=mixes, **special)
        self.o = MergedLinear(h * dv, [width])

    def forward(self, x: torch.Tensor, positions: torch.Tensor, v_first) -> tuple[torch.Tensor, torch.Tensor]:
        """(the result, this layer's own values [T, G * vdim] as projected)"""
        proj = self.proj(x)
        return self.o(self.attn(proj, positions, v_first=v_first)), proj[:, self.sizes[0] + self.sizes[1]:]


class MopalornFeedForward(nn.Module):
    def __init__(self, width: int, ff: int):
        super().__init__()
        self.up, self.down = MergedLinear(width, [ff]), MergedLinear(ff, [width])
        self.act = XIELU()

    def forward(self, x: torch.Tensor) -> torch.Tensor:
        return self.down(self.act(self.up(x)))


class MopalornLayer(nn.Module):
    def __init__(self, width: int, spec, eps: float, mixes: bool):
        super().__init__()
        kind, mixer, mlp = _get(spec, "type"), _get(spec, "mixer"), _get(spec, "mlp")
        if kind == "latent_attention":
            self.mixer = MopalornLatentAttention(width, mixer, eps)
        elif kind in ("attention", "attention_2"):
            self.mixer = MopalornAttention(width, mixer, kind == "attention_2", mixes)
        else:
            raise ValueError(f"unknown mixer type {kind!r}")
        self.norm1, self.norm1b = StreamNorm(width, eps, "rms"), StreamNorm(width, eps, "rms")
        self.mlp = None
        if mlp:
            if _get(mlp, "kind", "dense") != "dense":
                raise ValueError(f"unknown feed-forward kind {_get(mlp, 'kind')!r}")
            self.mlp = MopalornFeedForward(width, int(_get(mlp, "ff")))
            self.norm2, self.norm2b = StreamNorm(width, eps, "rms"), StreamNorm(width, eps, "rms")


class MopalornForCausalLM(nn.Module):
    requires_cache = True            # attention reads its keys from the paged cache in every step (no packed mode)
    supported_dtypes = (torch.bfloat16, torch.float32)

    def __init__(self, config) -> None:
        super().__init__()
        self.config = config
        width, vocab = int(config.width), int(config.vocab)
        eps = float(_get(config.norm, "eps", 1e-6))
        self.width, self.vocab, self.eps = width, vocab, eps
        self.logit_scale = float(getattr(config, "logit_scale", 1.0))
        self.embed = MergedLinear(width, [vocab])            # [vocab, width]: the token table and the output projection
        mixing = [i for i, spec in enumerate(config.layers) if self._mixes(spec)]
        self.first_mixing = mixing[0] if mixing else None    # the layer whose values the later ones mix in
        for i in mixing[1:]:
            assert self._value_sizes(config.layers[i]) == self._value_sizes(config.layers[mixing[0]]), f"layers {mixing[0]} and {i} mix values of different sizes"
        self.layers = nn.ModuleList([MopalornLayer(width, spec, eps, i in mixing[1:]) for i, spec in enumerate(config.layers)])
        self.final_norm = StreamNorm(width, eps, "rms")
        self.collect = None          # a list: receives a copy of the stream after every layer (debugging, tests)

    @staticmethod
    def _mixes(spec) -> bool:
        return _get(spec, "type") != "latent_attention" and bool(_get(_get(spec, "mixer"), "v_mix", False))

    @staticmethod
    def _value_sizes(spec) -> int:
        m = _get(spec, "mixer")
        return int(_get(m, "kv_heads", _get(m, "heads"))) * int(_get(m, "vdim", _get(m, "dim")))

    # ------------------------------------------------------------------ checkpoint names
    def weight_target(self, name: str):
        """(parameter name, shard id | None) of a checkpoint tensor; (None, None) for one that is stored and not used."""
        top = {"embed": "embed.weight", "final.norm": "final_norm.weight"}
        if name in top:
            return top[name], None
        m = re.fullmatch(r"l(\d+)\.(.+)", name)
        if not m or int(m.group(1)) >= len(self.layers):
            raise KeyError(f"checkpoint tensor {name!r} matches no parameter of the model")
        i, rest = int(m.group(1)), m.group(2)
        p, layer = f"layers.{i}.", self.layers[i]
        if rest in ("norm1", "norm1b"):
            return p + rest + ".weight", None
        if rest in ("norm2", "norm2b"):
            return (p + rest + ".weight", None) if layer.mlp is not None else (None, None)
        if rest.startswith("mlp.") and layer.mlp is not None:
            direct = {"up": "mlp.up.weight", "down": "mlp.down.weight", "act": "mlp.act.params"}
            if rest[4:] in direct:
                return p + direct[rest[4:]], None
        elif rest.startswith("mix."):
            leaf, mixer, pm = rest[4:], layer.mixer, p + "mixer."
            if leaf == "o":
                return pm + "o.weight", None
            if leaf in mixer.proj.shard_ids:
                return pm + "proj.weight", leaf
            if isinstance(mixer, MopalornLatentAttention):
                direct = {"dkv.norm": "attn.kv_norm", "uk": "attn.uk_t", "uv": "attn.uv"}
                if leaf in direct:
                    return pm + direct[leaf], None
            elif leaf == "sink" and mixer.attn.sinks is not None:
                return pm + "attn.sinks", None
            elif leaf == "vmix":                             # (the layer whose values are mixed in stores one without a use for it)
                return (pm + "attn.v_mix", None) if mixer.attn.v_mix is not None else (None, None)
        raise KeyError(f"checkpoint tensor {name!r} matches no parameter of the model")

    @staticmethod
    def synthetic_tensors(config, seed: int = 0, std: float = 0.02, device="cuda", dtype=torch.bfloat16):
        """Random weights in checkpoint naming (for benchmarks and smoke runs without a checkpoint)."""
        width, vocab = int(config.width), int(config.vocab)

        def mat(name, *shape, scale=std, shift=0.0):
            g = torch.Generator(device=device)
            g.manual_seed((zlib.crc32(name.encode()) ^ (seed * 0x9E3779B1)) & 0x7FFFFFFF)
            return name, (torch.randn(tuple(shape), generator=g, device=device, dtype=torch.float32) * scale + shift).to(dtype)

        yield mat("embed", vocab, width, scale=1.0)
        yield mat("final.norm", width, scale=0.1, shift=1.0)
        for i, spec in enumerate(config.layers):
            p, m, kind, mlp = f"l{i}.", _get(spec, "mixer"), _get(spec, "type"), _get(spec, "mlp")
            for n in ("norm1", "norm1b") + (("norm2", "norm2b") if mlp else ()):
                yield mat(p + n, width, scale=0.1, shift=1.0)
            h, d = int(_get(m, "heads")), int(_get(m, "dim"))
            dv = int(_get(m, "vdim", d))
            if kind == "latent_attention":
                dr, rank = int(_get(m, "rot_dim", 0) or 0), int(_get(m, "kv_rank"))
                yield mat(p + "mix.q", h * (d + dr), width)
                yield mat(p + "mix.dkv", rank + dr, width)
                yield mat(p + "mix.dkv.norm", rank, scale=0.1, shift=1.0)
                yield mat(p + "mix.uk", h * d, rank)
                yield mat(p + "mix.uv", h * dv, rank)
                yield mat(p + "mix.g", h * dv, width)
            else:
                g = int(_get(m, "kv_heads", h))
                for leaf, n in (("q", h * d), ("k", g * d), ("v", g * dv)):
                    yield mat(p + "mix." + leaf, n, width)
                if kind == "attention_2":
                    yield mat(p + "mix.sink", h, scale=1.0)
                if MopalornForCausalLM._mixes(spec):
                    yield mat(p + "mix.vmix", scale=0.1, shift=0.4)
            yield mat(p + "mix.o", width, h * dv)
            if mlp:
                ff = int(_get(mlp, "ff"))
                yield mat(p + "mlp.up", ff, width)
                yield mat(p + "mlp.down", width, ff)
                yield mat(p + "mlp.act", 2, scale=0.3)

    # ------------------------------------------------------------------ forward
    def forward(self, input_ids: torch.Tensor, positions: torch.Tensor) -> torch.Tensor:
        """The fp32 residual stream [T, width] after the last layer (the final norm runs on the rows that are projected)."""
        x = ops.embedding_pos_stream(input_ids, positions, self.embed.weight.data, None, 1.0)
        h = self.layers[0].norm1(x)
        v_first, last = None, len(self.layers) - 1

        def close(result, after, opening):
            """x += after(result); the opening norm of the next sublayer of the new x (None behind the last)"""
            spec = opening.spec() if opening is not None else {}
            return ops.residual_norm(x, a=result, a_weight=after.weight.data, branch_eps=after.eps, **spec)

        for i, layer in enumerate(self.layers):
            y, values = layer.mixer(h, positions, v_first)
            if i == self.first_mixing:
                v_first = values
            opening = self.layers[i + 1].norm1 if i < last else None
            h = close(y, layer.norm1b, layer.norm2 if layer.mlp is not None else opening)
            if layer.mlp is not None:
                h = close(layer.mlp(h), layer.norm2b, opening)
            if self.collect is not None:
                self.collect.append(x.clone())
        return x

    def gather_rows(self, hidden: torch.Tensor, rows: torch.Tensor) -> torch.Tensor:
        return ops.gather_rows_f32(hidden, rows)

    def compute_logits_rows(self, rows: torch.Tensor) -> torch.Tensor:
        """fp32 logits [R, vocab] of selected rows of the stream: final norm, the embedding table, scale."""
        return ops.logits_scale(self.embed(self.final_norm(rows), out_f32=True), self.logit_scale)

    def compute_logits(self, hidden: torch.Tensor) -> torch.Tensor:
        return self.compute_logits_rows(hidden)
