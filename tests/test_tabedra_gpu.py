"""Tabedra through the engine against the plain float64 restatement in tests/tabedra_reference.py.

Every test makes its own small configuration and random weights (written as config.json + model.safetensors into a
temporary directory, so the config reader and the loader are part of what is tested), runs a schedule through
nanovllm.trace_replay.TraceReplay (the engine's runner, page and slot manager and kernels) and compares logits - and, for
single layers, the sum of the residual streams - with the reference run over each whole sequence.  fp32 serving is compared
tightly, bf16 serving within the rounding of its products; the bf16 weights route calmly (the correction decides which
experts are chosen, the scores how they are weighted), so that rounding does not turn a close choice round.
"""
import copy
import json
import math
import os

import numpy as np
import pytest
import torch

import tabedra_reference as R

pytestmark = pytest.mark.gpu

MOE_A = {"kind": "moe", "expert": {"ff": 40}, "router": {"experts": 6, "top": 2}, "shared": {"ff": 56}}
MOE_B = {"kind": "moe", "expert": {"ff": 21}, "router": {"experts": 5, "top": 3}, "shared": {"ff": 30}}
# sizes of the matrix-core attention in bf16 (multiples of 16), a window edge inside the test lengths, distances beyond the bias table's reach
ATT_A = {"type": "attention", "mlp": MOE_A,
         "mixer": {"heads": 4, "kv_heads": 2, "dim": 32, "vdim": 16, "conv": 4, "scale": 0.2, "bias_max": 30, "mask": {"size": 43}}}
ATT_B = {"type": "attention", "mlp": None,
         "mixer": {"heads": 2, "kv_heads": 2, "dim": 48, "vdim": 48, "conv": 2, "scale": 0.15, "bias_max": 90, "mask": {"size": 20}}}
# sizes that no tile divides (the vector-ALU attention in both types), a convolution wider than most portions
ATT_C = {"type": "attention", "mlp": MOE_B,
         "mixer": {"heads": 6, "kv_heads": 2, "dim": 10, "vdim": 14, "conv": 5, "scale": 0.3, "bias_max": 25, "mask": {"size": 33}}}
ATT_D = {"type": "attention", "mlp": None,
         "mixer": {"heads": 3, "kv_heads": 1, "dim": 16, "vdim": 32, "conv": 1, "scale": 0.4, "bias_max": 17, "mask": {"size": 61}}}


def shared(layer, j, **changes):
    """The layer with the keys and values of layer j (and changes of what is its own)."""
    return dict(copy.deepcopy(layer), mixer=dict(copy.deepcopy(layer["mixer"]), kv_from=j, **changes))


def config(layers, width=96, vocab=131, streams=3, eps=1e-5, bias_rows=16, buckets=97):
    return {"architecture": "Tabedra", "vocab": vocab, "width": width, "max_positions": 1400, "streams": streams, "norm": {"eps": eps},
            "embedding": {"bigram": {"buckets": buckets, "mul_prev": 13, "mul_cur": 5}}, "layers": copy.deepcopy(layers), "_rows": bias_rows}


CFG_MIX = config([ATT_A, ATT_C, shared(ATT_A, 0, mask={"size": 60}, bias_max=44, scale=0.3), ATT_B])
CFG_FLAT = config([ATT_B, shared(ATT_B, 0, conv=3), ATT_D, shared(ATT_D, 2)], width=128, vocab=200, streams=2, eps=1e-6, bias_rows=8, buckets=50)


def random_weights(cfg: dict, seed: int, calm: bool = False) -> dict:
    """bf16 weights in checkpoint naming.  `calm`: corrections far apart beside scores close to each other."""
    g = torch.Generator().manual_seed(seed)
    D, V, S = cfg["width"], cfg["vocab"], cfg["streams"]
    W = {}

    def mat(name, out, inp, scale=1.0):
        W[name] = torch.randn(out, inp, generator=g) * (scale / math.sqrt(inp))

    def vec(name, n, scale=0.2, shift=1.0):
        W[name] = shift + scale * torch.randn(n, generator=g)

    W["embed"] = torch.randn(V, D, generator=g)
    W["pos"] = torch.randn(cfg["max_positions"], D, generator=g) * 0.3
    W["bigram"] = torch.randn(cfg["embedding"]["bigram"]["buckets"] + 1, D, generator=g) * 0.7
    vec("final.norm", D)
    vec("final.norm.b", D, shift=0.0)
    mat("head", V, D)
    for i, L in enumerate(cfg["layers"]):
        p, m, mlp = f"l{i}.", L["mixer"], L.get("mlp")
        for q in (1, 2) if mlp else (1,):
            vec(p + f"norm{q}", D)
            vec(p + f"norm{q}.b", D, shift=0.0)
            vec(p + f"hc{q}.in", S, 0.3, 1.0 / S)
            vec(p + f"hc{q}.out", S, 0.4, 0.8)
            W[p + f"hc{q}.mix"] = torch.eye(S) * 0.8 + 0.25 * torch.randn(S, S, generator=g)
        h, kv, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        for leaf, n in [("q", h * d)] + ([("k", kv * d), ("v", kv * dv)] if m.get("kv_from") is None else []):
            mat(p + "mix." + leaf, n, D)
            W[p + f"mix.{leaf}.conv"] = torch.randn(n, m["conv"], generator=g) * 0.6
        W[p + "mix.rel"] = torch.randn(cfg["_rows"], h, generator=g)
        mat(p + "mix.g", h * dv, D)
        mat(p + "mix.o", D, h * dv, 2.0)
        if mlp:
            E, ff = mlp["router"]["experts"], mlp["expert"]["ff"]
            for e in range(E):
                mat(p + f"mlp.e{e}.up", ff, D)
                mat(p + f"mlp.e{e}.down", D, ff)
            mat(p + "mlp.router", E, D, 0.4 if calm else 1.5)
            W[p + "mlp.correction"] = torch.randperm(E, generator=g).float() * 0.5 if calm else torch.randn(E, generator=g) * 0.2
            if mlp.get("shared"):
                mat(p + "mlp.shared.up", mlp["shared"]["ff"], D)
                mat(p + "mlp.shared.down", D, mlp["shared"]["ff"])
    return {k: v.to(torch.bfloat16) for k, v in W.items()}


def write_model(path, cfg: dict, weights: dict) -> str:
    from safetensors.torch import save_file
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump({k: v for k, v in cfg.items() if not k.startswith("_")}, f)
    save_file({k: v.contiguous() for k, v in weights.items()}, os.path.join(path, "model.safetensors"))
    return str(path)


class Case:
    """A model on disk, its reference weights and cached reference logits per token list."""

    def __init__(self, tmp, cfg, seed=0, weights=None, calm=False):
        self.cfg = cfg
        w = weights if weights is not None else random_weights(cfg, seed, calm)
        self.path = write_model(tmp, cfg, w)
        self.W = {k: v.double() for k, v in w.items()}
        self._ref = {}

    def ref(self, tokens):
        key = tuple(tokens)
        if key not in self._ref:
            self._ref[key] = R.forward(self.W, self.cfg, list(tokens)).numpy()
        return self._ref[key]

    def replay(self, dtype="float32", max_tokens=2048, slots=4):
        from nanovllm.trace_replay import TraceReplay
        return TraceReplay(self.path, dtype, max_tokens, slots)


def tokens_of(cfg, n, seed):
    return torch.randint(0, cfg["vocab"], (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def rel_err(got, want):
    """Largest row error, mean removed, relative to the spread of the reference logits."""
    d = got - want
    d = d - d.mean(-1, keepdims=True)
    return float(np.sqrt((d ** 2).mean(-1)).max() / want.std())


TOL = {"float32": 1e-4, "bfloat16": 8e-2}


@pytest.fixture(scope="module")
def mix_case(tmp_path_factory):
    cases = {dt: Case(tmp_path_factory.mktemp("tabedra_mix"), CFG_MIX, seed=1, calm=dt == "bfloat16") for dt in TOL}
    return lambda dtype="float32": cases[dtype]


@pytest.fixture(scope="module")
def flat_case(tmp_path_factory):
    case = Case(tmp_path_factory.mktemp("tabedra_flat"), CFG_FLAT, seed=2)      # (no experts: nothing to route)
    return case


def run_schedule(rp, case, requests: dict, schedule: list, dtype: str, tol=None):
    """schedule: list of steps, each a list of (request id, token count); every position's logits are asked for and
    compared with the reference of the whole request.  Requests end when their tokens are used up."""
    at = {r: 0 for r in requests}
    for step in schedule:
        entries, spans, end = [], [], []
        for rid, count in step:
            lo, hi = at[rid], at[rid] + count
            entries.append({"id": rid, "tokens": requests[rid][lo:hi], "want": list(range(count))})
            spans.append((rid, lo, hi))
            at[rid] = hi
            if hi == len(requests[rid]):
                end.append(rid)
        got = rp.step(entries, end)
        row = 0
        for rid, lo, hi in spans:
            err = rel_err(got[row:row + hi - lo], case.ref(requests[rid])[lo:hi])
            assert err < (tol or TOL[dtype]), f"request {rid} tokens {lo}..{hi}: error {err:.3g}"
            row += hi - lo
    assert all(at[r] == len(requests[r]) for r in requests)


# ----------------------------------------------------------------------------------------------------- single mechanisms
@pytest.mark.parametrize("layer", [ATT_A, ATT_B, ATT_C, ATT_D], ids=["matrix cores in bf16", "no feed-forward", "ragged", "one tap"])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_one_layer_stream_matches(tmp_path, layer, dtype):
    """One layer of each kind: the sum of the streams after it and the logits; 80 tokens cross every window and the bias tables' reach."""
    cfg = config([layer], width=72, vocab=50)
    case = Case(tmp_path, cfg, seed=3, calm=dtype == "bfloat16")
    toks = tokens_of(cfg, 80, 5)
    rp = case.replay(dtype)
    try:
        rp.runner.model.collect = []
        got = rp.step([{"id": 0, "tokens": toks, "want": list(range(len(toks)))}], [0])
        stream = rp.runner.model.collect[0].cpu().numpy()
    finally:
        rp.close()
    col = []
    want = R.forward(case.W, cfg, toks, col).numpy()
    assert np.abs(stream - col[0].numpy()).max() < (1e-4 if dtype == "float32" else 0.1) * max(1.0, float(col[0].abs().max()))
    assert rel_err(got, want) < TOL[dtype]


def test_every_layer_of_a_stack(mix_case):
    case = mix_case()
    toks = tokens_of(CFG_MIX, 70, 7)
    rp = case.replay("float32")
    try:
        rp.runner.model.collect = []
        rp.step([{"id": 0, "tokens": toks, "want": [0]}], [0])
        streams = [c.cpu().numpy() for c in rp.runner.model.collect]
    finally:
        rp.close()
    col = []
    R.forward(case.W, CFG_MIX, toks, col)
    assert len(streams) == len(col) == 4
    for n, (a, b) in enumerate(zip(streams, col)):
        assert np.abs(a - b.numpy()).max() < 1e-4 * max(1.0, float(b.abs().max())), f"layer {n}"


def test_distance_buckets_against_their_formula():
    from nanovllm.layers.attention import WindowedBiasAttention
    for rows, reach in [(2, 5), (4, 3), (8, 17), (16, 30), (32, 100), (32, 129), (64, 1000), (10, 77)]:
        got = WindowedBiasAttention.distance_buckets(rows, reach)
        for n in range(2 * reach):
            assert got[min(n, len(got) - 1)] == R.bucket(n, rows, reach), (rows, reach, n)
        assert got[-1] == rows - 1 and got.count(rows - 1) == 1
        for window in (1, rows // 2, rows // 2 + 1, reach, reach + 9):
            assert WindowedBiasAttention.distance_buckets(rows, reach, window) == got[:window]
    # edges that the logarithms hit exactly: bucket 4 + m begins at 4 * 2^m
    assert [WindowedBiasAttention.distance_buckets(8, 64).index(b) for b in (4, 5, 6, 7)] == [4, 8, 16, 32]
    with pytest.raises(AssertionError):
        WindowedBiasAttention.distance_buckets(16, 8)


def paged(x, pages, page, transposed):
    """[T, G, d] -> page cache [n, page, G, d] (or [n, G, d, page]) through the page list."""
    T, G, d = x.shape
    cache = torch.zeros(8, G, d, page, dtype=x.dtype) if transposed else torch.zeros(8, page, G, d, dtype=x.dtype)
    for t in range(T):
        if transposed:
            cache[pages[t // page], :, :, t % page] = x[t]
        else:
            cache[pages[t // page], t % page] = x[t]
    return cache


@pytest.mark.parametrize("H,G,d,dv,window,rows,reach", [(4, 2, 32, 32, 40, 16, 30), (6, 3, 48, 16, 0, 32, 100), (6, 2, 20, 12, 33, 8, 50), (2, 2, 64, 64, 1, 4, 9),
                                                        (40, 2, 16, 16, 50, 8, 300), (3, 1, 80, 112, 0, 32, 500), (2, 1, 128, 128, 200, 64, 150), (16, 1, 16, 32, 0, 32, 9000),
                                                        (1, 1, 256, 256, 0, 2, 3), (2, 2, 48, 48, 20, 16, 90), (2, 1, 80, 80, 90, 16, 40), (4, 1, 96, 96, 60, 16, 70), (2, 1, 192, 192, 0, 8, 33), (3, 1, 144, 208, 70, 16, 50)])
def test_attention_with_a_distance_bias_and_an_element_gate(H, G, d, dv, window, rows, reach):
    """Prompts, portions and one-query steps (where, in bf16, a group's heads share a workgroup and the key tiles go to several) over two
    sequences on scattered pages; matrix-core sizes and others, tables that end inside and beyond the context, one that does not fit
    beside its group's others in LDS."""
    from nanovllm import ops
    from nanovllm.layers.attention import WindowedBiasAttention
    g = torch.Generator().manual_seed(6)
    page = 256
    rel = torch.randn(rows, H, generator=g) * 2
    bias = rel[torch.tensor(WindowedBiasAttention.distance_buckets(rows, reach, window))].t().contiguous().cuda()
    for cast, tol in ((torch.float32, 1e-4), (torch.bfloat16, 3e-2)):
        lens, pages = [620, 70], [[4, 0, 2], [1, 0, 0]]
        q, k, v = ([torch.randn(n, hh, dd, generator=g).to(cast) for n in lens] for hh, dd in ((H, d), (G, d), (G, dv)))
        logits = [torch.randn(n, 3 + H * dv, generator=g).to(cast) * 2 for n in lens]
        kc, vc = (sum(paged(x[b], pages[b], page, tr) for b in range(2)).cuda() for x, tr in ((k, False), (v, True)))
        tables = torch.tensor(pages, dtype=torch.int32).cuda()
        for take in ((40, 70), (1, 1), (130, 2), (1, 5)):
            for gated in (True, False):
                ends = [lens[0] - (5 if take[0] == 1 else 0), lens[1] - (9 if take[1] == 1 else 0)]
                cut = lambda x: torch.cat([x[b][ends[b] - take[b]:ends[b]].reshape(take[b], -1) for b in range(2)]).cuda()
                cu = torch.tensor([0, take[0], take[0] + take[1]], dtype=torch.int32).cuda()
                out = ops.attn_paged_any(cut(q), kc, vc, None if take == (1, 1) else cu, torch.tensor(ends, dtype=torch.int32).cuda(), tables, 0.2, H, G, d, dv,
                                         window=window, bias=bias, gate_elems=cut(logits)[:, 3 if d % 16 else 0:][:, :H * dv] if gated else None).cpu().double().view(-1, H, dv)
                row = 0
                for b in range(2):
                    some = [i for i in range(ends[b] - take[b], ends[b]) if i % 17 == 3 or i >= ends[b] - 2]     # (a sample of the rows keeps the oracle quick)
                    n = ends[b]
                    ref = R.attend(q[b][:n].double(), k[b][:n].double(), v[b][:n].double(), 0.2, rel.double(), reach, window, some)
                    if gated:
                        ref = ref * torch.sigmoid(logits[b][:n, 3 if d % 16 else 0:][:, :H * dv].double()).view(n, H, dv)
                    for i in some:
                        got = out[row + i - (n - take[b])]
                        assert (got - ref[i]).abs().max() < tol * max(1.0, float(ref[i].abs().max())), (cast, take, gated, b, i)
                    row += take[b]


def test_bias_beside_other_options_takes_the_general_kernel():
    """A distance bias together with a softcap, sinks, kept first tokens: against the formula in both types."""
    from nanovllm import ops
    g = torch.Generator().manual_seed(4)
    H, d, n = 2, 16, 90
    bias = torch.randn(H, 20, generator=g)
    for cast, tol in ((torch.float32, 1e-4), (torch.bfloat16, 3e-2)):
        q, k, v = (torch.randn(n, H, d, generator=g).to(cast) for _ in range(3))
        out = ops.attn_paged_any(q.reshape(n, -1).cuda(), paged(k, [3], 256, False).cuda(), paged(v, [3], 256, True).cuda(), torch.tensor([0, n], dtype=torch.int32).cuda(),
                                 torch.tensor([n], dtype=torch.int32).cuda(), torch.tensor([[3]], dtype=torch.int32).cuda(), 0.4, H, H, d, d, window=30, keep_first=2,
                                 softcap=2.0, bias=bias.cuda(), sinks=torch.tensor([0.5, -1.0]).cuda()).cpu().double().view(n, H, d)
        for i in range(0, n, 7):
            for h in range(H):
                seen = [j for j in range(i + 1) if i - j < 30 or j < 2]
                s = torch.stack([2.0 * torch.tanh((q[i, h].double() @ k[j, h].double()) * 0.4 / 2.0) + bias[h, min(i - j, 19)].double() for j in seen])
                e = torch.exp(s)
                want = (e[:, None] * v[seen, h].double()).sum(0) / (e.sum() + math.exp([0.5, -1.0][h]))
                assert (out[i, h] - want).abs().max() < tol * 3, (cast, i, h)


@pytest.mark.parametrize("H,G,d,dv,taps", [(4, 2, 32, 16, 4), (3, 1, 10, 14, 3), (2, 2, 64, 96, 2), (1, 1, 200, 130, 6), (5, 1, 8, 8, 1), (2, 1, 5, 3, 9), (2, 1, 128, 128, 0), (1, 1, 512, 264, 3)])
def test_convolved_queries_keys_and_values(H, G, d, dv, taps):
    """nvh_attn_conv_prep over steps that mix portions and single tokens, continue in slots, start on slots that others left and skip padded
    rows: every row against the convolution of the whole sequence; one-token steps bring the state up to date by themselves.  More
    than 512 tokens take the wide tile."""
    from nanovllm import ops
    g = torch.Generator().manual_seed(9)
    page, eps, C = 256, 1e-5, H * d + G * (d + dv)
    for cast, tol in ((torch.float32, 2e-5), (torch.bfloat16, 3e-2)):
        for own in (True, False):
            ch = C if own else H * d
            w = (torch.randn(ch, taps, generator=g) * 0.6).to(cast) if taps else None
            lens = [9, 700, 40]
            rows = [torch.randn(n, ch + 5, generator=g).to(cast) for n in lens]
            plain = [R.causal_conv(x[:, :ch].double(), w.double()) if taps else x[:, :ch].double() for x in rows]
            state = torch.full((3, max(taps - 1, 1), ch), 7.0).cuda()                 # (what others left behind)
            kc, vc = torch.zeros(9, page, G, d, dtype=cast).cuda(), torch.zeros(9, G, dv, page, dtype=cast).cuda()
            pages = [[8], [0, 3, 5], [6]]
            at = [0, 0, 0]
            for take in ([3, 2, 1], [1, 1, 1], [0, 600, 0], [2, 1, 30], [1, 1, 1], [1, 1, 1], [0, 40, 2]):
                live = [b for b in range(3) if take[b]]
                n = [take[b] for b in live]
                ctx = torch.tensor([at[b] + take[b] for b in live], dtype=torch.int32)
                cu = torch.tensor([0] + list(np.cumsum(n)), dtype=torch.int32)
                proj = torch.cat([rows[b][at[b]:at[b] + take[b]] for b in live])
                slot = torch.tensor([pages[b][p // page] * page + p % page for b in live for p in range(at[b], at[b] + take[b])], dtype=torch.int32)
                slots = torch.tensor([2 - b for b in live], dtype=torch.int32)
                single = all(x == 1 for x in n)
                if single:                                                           # as a captured step: a padded row behind the real ones
                    proj, ctx = torch.cat([proj, torch.ones(1, ch + 5, dtype=cast)]), torch.cat([ctx, torch.zeros(1, dtype=torch.int32)])
                    slot, slots = torch.cat([slot, torch.tensor([-1], dtype=torch.int32)]), torch.cat([slots, torch.tensor([-1], dtype=torch.int32)])
                q = ops.attn_conv_prep(proj.cuda(), None if w is None else w.cuda(), state if taps > 1 else None, slots.cuda(), None if single else cu.cuda(), ctx.cuda(),
                                       slot.cuda(), kc if own else None, vc if own else None, H, G, d, dv, eps).cpu().double()
                row = 0
                for b in live:
                    for p in range(at[b], at[b] + take[b]):
                        want = R.unit(plain[b][p, :H * d].view(H, d), eps).reshape(-1)
                        assert (q[row] - want).abs().max() < tol * max(1.0, float(want.abs().max())), (cast, own, take, b, p)
                        row += 1
                    at[b] += take[b]
                    if taps > 1:
                        for s in range(taps - 1):
                            p = at[b] - taps + 1 + s
                            want = rows[b][p, :ch].float() if p >= 0 else torch.zeros(ch)
                            assert torch.equal(state[2 - b, s].cpu(), want), (cast, take, b, s)
            if own:
                kcpu, vcpu = kc.cpu().double(), vc.cpu().double()
                for b in range(3):
                    for p in range(at[b]):
                        pg, off = pages[b][p // page], p % page
                        want = R.unit(plain[b][p, H * d:(H + G) * d].view(G, d), eps)
                        assert (kcpu[pg, off] - want).abs().max() < tol * max(1.0, float(want.abs().max())), (cast, b, p)
                        want = plain[b][p, (H + G) * d:].view(G, dv)
                        assert (vcpu[pg, :, :, off] - want).abs().max() < tol * max(1.0, float(want.abs().max())), (cast, b, p)
                assert int((kcpu != 0).any(-1).any(-1).sum()) == sum(at)             # nothing else is touched


def test_streams_close_and_open_against_their_formula():
    """x_t <- sum_s mix[s, t] x_s + out[t] y with y of every kind, then the norm of the next weighted sum; stream counts and widths of both forms."""
    from nanovllm import ops
    g = torch.Generator().manual_seed(3)
    for S in (1, 2, 3, 4, 5, 16):
        for dim in (50, 96, 1024, 2052, 8192) if S in (2, 4) else (36, 1030):
            T, top = 5, 2
            x, a, c = torch.randn(T, S, dim, generator=g) * 3, torch.randn(T, dim, generator=g), torch.randn(T, dim, generator=g)
            pairs, wts = torch.randn(T * top, dim, generator=g), torch.rand(T, top, generator=g)
            pos = torch.randperm(T * top, generator=g).int()
            mix, out, inn = torch.randn(S, S, generator=g), torch.randn(S, generator=g), torch.randn(S, generator=g)
            nw, nb = torch.randn(dim, generator=g), torch.randn(dim, generator=g)
            for cast in (torch.float32, torch.bfloat16):
                tol = 3e-5 if cast == torch.float32 else 2e-2
                ac, pc, wc, bc = (z.to(cast) for z in (a, pairs, nw, nb))
                for terms in ("a", "c32", "pairs", "a pairs", "none"):
                    y = torch.zeros(T, dim, dtype=torch.float64)
                    kw = {}
                    if "a" in terms.split():
                        y, kw["a"] = y + ac.double(), ac.cuda()
                    if "c32" in terms:
                        y, kw["c32"] = y + c.double(), c.cuda()
                    if "pairs" in terms:
                        y = y + torch.stack([sum(wts[t, r].double() * pc[int(pos[t * top + r])].double() for r in range(top)) for t in range(T)])
                        kw.update(pairs=pc.cuda(), plan=dict(pos_of_pair=pos.cuda(), pairs=T * top), weights=wts.cuda())
                    want = torch.stack([sum(mix[s, t].double() * x[:, s].double() for s in range(S)) + out[t].double() * y for t in range(S)], 1)
                    if terms == "none":
                        want = x.double()
                    u = sum(inn[t].double() * want[:, t] for t in range(S))
                    xg = x.cuda()
                    streams = {} if terms == "none" else dict(mix=mix.cuda(), out_weights=out.cuda())
                    h = ops.hyper_norm(xg, **streams, in_weights=inn.cuda(), **kw, norm="layer", weight=wc.cuda(), bias=bc.cuda(), eps=1e-3)
                    assert (xg.cpu().double() - want).abs().max() < 3e-5 * float(want.abs().max()), (S, dim, terms)
                    ref = R.layer_norm(u, wc.double(), bc.double(), 1e-3)
                    assert h.dtype == cast and (h.cpu().double() - ref).abs().max() < tol * float(ref.abs().max()), (S, dim, cast, terms)
                    xg = x.cuda()
                    h = ops.hyper_norm(xg, **streams, **kw, norm="rms", weight=wc.cuda(), eps=1e-3)                  # (ones: the plain sum)
                    ref = R.unit(want.sum(1), 1e-3) * wc.double()
                    assert (h.cpu().double() - ref).abs().max() < tol * float(ref.abs().max()), (S, dim, cast, terms)
                    if terms != "none":
                        xg = x.cuda()
                        assert ops.hyper_norm(xg, **streams, in_weights=inn.cuda(), **kw) is None
                        assert (xg.cpu().double() - want).abs().max() < 3e-5 * float(want.abs().max())


def test_bigram_rows_and_the_last_token_of_every_sequence():
    from nanovllm import ops
    g = torch.Generator().manual_seed(8)
    for dim, S in ((40, 3), (37, 2), (1100, 1)):
        V, B = 300, 61
        table, pos_t, big = (torch.randn(n, dim, generator=g) for n in (V, 500, B + 1))
        spec = {"buckets": B, "mul_prev": 1009, "mul_cur": 77}
        seqs = [torch.randint(0, V, (n,), generator=g).tolist() for n in (30, 8, 5)]
        for cast in (torch.float32, torch.bfloat16):
            tc, pc, bc = (z.to(cast) for z in (table, pos_t, big))
            last = torch.full((4,), 123, dtype=torch.int32).cuda()
            at = [0, 0, 0]
            for take in ([5, 1, 0], [1, 1, 1], [2, 0, 1], [1, 1, 1], [21, 5, 2]):
                live = [b for b in range(3) if take[b]]
                ids = [t for b in live for t in seqs[b][at[b]:at[b] + take[b]]]
                positions = [p for b in live for p in range(at[b], at[b] + take[b])]
                ctx = [at[b] + take[b] for b in live]
                slots = [3 - b for b in live]
                cu = torch.tensor([0] + list(np.cumsum([take[b] for b in live])), dtype=torch.int32)
                single = take == [1, 1, 1]
                if single:                                                           # (a padded row)
                    ids, positions, ctx, slots = ids + [7], positions + [0], ctx + [0], slots + [-1]
                x = ops.embedding_bigram_stream(torch.tensor(ids).cuda(), torch.tensor(positions).cuda(), tc.cuda(), S, pc.cuda(), bc.cuda(), 1009, 77, last,
                                                torch.tensor(slots, dtype=torch.int32).cuda(), None if single else cu.cuda(), torch.tensor(ctx, dtype=torch.int32).cuda()).cpu().double()
                row = 0
                for b in live:
                    for p in range(at[b], at[b] + take[b]):
                        t = seqs[b][p]
                        want = tc[t].double() + bc[R.bigram_row(seqs[b][p - 1] if p else None, t, spec)].double() + pc[p].double()
                        assert (x[row] - want).abs().max() < 1e-5, (take, b, p)
                        row += 1
                    at[b] += take[b]
                    assert int(last[3 - b]) == seqs[b][at[b] - 1]
            assert int(last[0]) == 123


def test_routing_weights_divided_by_their_sum():
    from nanovllm import ops
    g = torch.Generator().manual_seed(2)
    for T, K, E, top in [(9, 64, 6, 2), (5, 50, 5, 5), (3, 96, 70, 1), (2, 64, 300, 8)]:
        x, w, corr = torch.randn(T, K, generator=g), torch.randn(E, K, generator=g) * 0.2, torch.randn(E, generator=g) * 0.1
        ids, weights, _ = ops.moe_route_scored(x.cuda(), w.cuda(), top, corr.cuda(), renorm=True)
        for t in range(T):
            want = R.route(w.double() @ x[t].double(), corr.double(), top)
            assert ids[t].tolist() == [e for e, _ in want]
            assert (weights[t].cpu().double() - torch.tensor([v for _, v in want], dtype=torch.float64)).abs().max() < 1e-5


def test_grouped_products_do_not_depend_on_how_many_rows_an_expert_has():
    """Few rows (16, 32 at most: operands straight from memory) and many (tiles through LDS): the same bits for the same row; the squared relu
    in the epilogue; against float64."""
    from nanovllm import ops
    g = torch.Generator().manual_seed(5)
    for N, K in [(72, 96), (200, 320), (64, 1024), (37, 50), (130, 33)]:
        for cast in (torch.float32, torch.bfloat16):
            T, E = 90, 4
            x, w = torch.randn(T, K, generator=g).to(cast), (torch.randn(E, N, K, generator=g) / math.sqrt(K)).to(cast)
            ids = torch.tensor([0] * 70 + [1] * 14 + [2] * 5 + [3] * 1, dtype=torch.int32)[:, None]
            for act in (None, "relu2"):
                plan = ops.moe_align(ids.cuda(), E)
                y = ops.linear_grouped(x.cuda(), w.cuda(), plan, gather=True, act=act)
                y = y[plan["pos_of_pair"].long()]
                want = torch.stack([w[int(ids[t])].double() @ x[t].double() for t in range(T)])
                want = torch.clamp(want, min=0.0) ** 2 if act else want
                assert (y.cpu().double() - want).abs().max() < (1e-4 if cast == torch.float32 else 0.12), (N, K, cast, act)
                for count in (1, 16, 17, 30, 33):                                    # the first `count` tokens alone with expert 0
                    few = ops.moe_align(torch.zeros(count, 1, dtype=torch.int32).cuda(), E)
                    z = ops.linear_grouped(x[:count].cuda(), w.cuda(), few, gather=True, act=act)[few["pos_of_pair"].long()]
                    assert torch.equal(z, y[:count]), (N, K, cast, act, count)


# ----------------------------------------------------------------------------------------------------- schedules
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_prefill_then_token_by_token(mix_case, dtype):
    toks = tokens_of(CFG_MIX, 100, 11)
    case = mix_case(dtype)
    rp = case.replay(dtype)
    try:
        run_schedule(rp, case, {"a": toks}, [[("a", 45)]] + [[("a", 1)]] * 55, dtype)
        # the first tokens of a sequence, one by one from the very start (one key, a convolution over nothing, no token before)
        run_schedule(rp, case, {"b": toks[:30]}, [[("b", 1)]] * 30, dtype)
    finally:
        rp.close()


def test_portions_of_every_size_give_the_same_logits(mix_case):
    toks = tokens_of(CFG_MIX, 100, 13)
    case = mix_case()
    rp = case.replay("float32")
    try:
        for sizes in ([100], [2] * 50, [3, 2, 17, 2, 33, 16, 2, 25], [64, 36], [1, 99], [22, 1, 1, 17, 2, 57], [4, 5, 3, 6, 2, 7, 73]):
            assert sum(sizes) == 100
            run_schedule(rp, case, {"a": toks}, [[("a", s)] for s in sizes], "float32")
    finally:
        rp.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_mixed_batches_of_unequal_requests(mix_case, dtype):
    reqs = {"a": tokens_of(CFG_MIX, 75, 21), "b": tokens_of(CFG_MIX, 9, 22), "c": tokens_of(CFG_MIX, 33, 23), "d": tokens_of(CFG_MIX, 2, 24)}
    sched = [[("a", 30), ("b", 3)], [("a", 1), ("b", 2), ("c", 20)], [("b", 1), ("a", 17), ("c", 1), ("d", 2)], [("c", 2), ("a", 27), ("b", 3)],
             [("c", 10)]]
    case = mix_case(dtype)
    rp = case.replay(dtype)
    try:
        run_schedule(rp, case, reqs, sched, dtype)
    finally:
        rp.close()


def test_pages_and_slots_are_used_again(flat_case):
    """A pool of three pages and two slots serves six requests one after another and in pairs: every request after the first two runs on pages
    and slots (convolution inputs, last token) that others have left behind."""
    reqs = {i: tokens_of(CFG_FLAT, n, 30 + i) for i, n in enumerate([300, 120, 257, 40, 256, 130])}
    rp = flat_case.replay("float32", max_tokens=256, slots=2)            # ceil(256/256) + 2 = 3 pages
    assert len(rp.scheduler.block_manager.blocks) == 3
    try:
        run_schedule(rp, flat_case, {0: reqs[0]}, [[(0, 200)], [(0, 100)]], "float32")
        run_schedule(rp, flat_case, {1: reqs[1], 2: reqs[2]}, [[(1, 100), (2, 7)], [(1, 20), (2, 250)]], "float32")
        run_schedule(rp, flat_case, {3: reqs[3], 4: reqs[4]}, [[(4, 255), (3, 39)], [(3, 1), (4, 1)]], "float32")
        run_schedule(rp, flat_case, {5: reqs[5]}, [[(5, 1)], [(5, 128)], [(5, 1)]], "float32")
        assert len(rp.scheduler.block_manager.free_block_ids) == 3
        run_schedule(rp, flat_case, {"again": reqs[0]}, [[("again", 300)]], "float32")
    finally:
        rp.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_page_borders_in_prompts_and_in_decoding(flat_case, dtype):
    """Portions that end one token before, at and after a page border, then decoding across the next one; portions that end around window
    edges."""
    toks = tokens_of(CFG_FLAT, 530, 41)
    rp = flat_case.replay(dtype, max_tokens=1100)
    try:
        run_schedule(rp, flat_case, {"a": toks}, [[("a", 255)], [("a", 1)], [("a", 1)], [("a", 2)], [("a", 251)], [("a", 3)]] + [[("a", 1)]] * 17, dtype)
        for first in (19, 20, 21, 60, 61, 62, 254, 256):
            run_schedule(rp, flat_case, {"b": toks[:first + 9]}, [[("b", first)], [("b", 7)], [("b", 1)], [("b", 1)]], dtype)
    finally:
        rp.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_one_token_steps_of_sequences_of_unequal_length(flat_case, dtype):
    """Steps in which every sequence brings one token; then fewer sequences as the short requests end."""
    reqs = {i: tokens_of(CFG_FLAT, n, 80 + i) for i, n in enumerate([12, 75, 135, 300])}
    first = {0: 2, 1: 64, 2: 129, 3: 290}
    sched = [[(i, first[i]) for i in reqs]] + [[(i, 1) for i in reqs if first[i] + k < len(reqs[i])] for k in range(11)]
    rp = flat_case.replay(dtype, max_tokens=1100)
    try:
        run_schedule(rp, flat_case, reqs, [st for st in sched if st], dtype)
    finally:
        rp.close()


def test_long_decoding(flat_case):
    toks = tokens_of(CFG_FLAT, 290, 43)
    rp = flat_case.replay("float32", max_tokens=512)
    try:
        run_schedule(rp, flat_case, {"a": toks}, [[("a", 5)]] + [[("a", 1)]] * 285, "float32")
    finally:
        rp.close()


# ----------------------------------------------------------------------------------------------------- faults that random weights would hide
ASKER, ASKED = 1, 2          # token ids: the query of ASKER scores high on the key of ASKED, all other scores are near zero


def asking_case(tmp, layers):
    """Heads that compare one coordinate: ASKED's key points along it, ASKER's query too, every other key and query along two others.
    Convolutions pass the token itself, the bigram table and all but the last layer's results are zero: what the last token sees of
    ASKED shows in its logits, and nothing else of ASKED does."""
    cfg = config(layers, width=64, vocab=700, streams=2)
    w = random_weights(cfg, 9)
    w["embed"][:, :3] = 0
    w["embed"][ASKED, 0] = w["embed"][ASKER, 1] = 20.0
    w["bigram"][:] = 0
    w["pos"][:, :3] = 0
    for i, layer in enumerate(cfg["layers"]):
        m, p = layer["mixer"], f"l{i}.mix."
        w[f"l{i}.norm1"][:3] = torch.tensor([1.0, 1.0, 0.0])
        w[f"l{i}.norm1.b"][:3] = torch.tensor([0.0, 0.0, 1.0])             # (a coordinate that is one for every token)
        w[f"l{i}.hc1.in"] = torch.tensor([0.5, 0.5]).to(torch.bfloat16)
        w[f"l{i}.hc1.mix"] = torch.eye(2).to(torch.bfloat16)
        for leaf, heads, marker, other in (("q", m["heads"], 1, 2), ("k", m["kv_heads"], 0, 1)):
            if p + leaf in w:
                x = torch.zeros(heads, m["dim"], 64)
                x[:, 0, marker] = 1.0
                x[:, other, 2] = 0.7
                w[p + leaf] = x.reshape(-1, 64).to(torch.bfloat16)
        for leaf in ("q", "k", "v"):
            if p + leaf in w:
                w[p + leaf + ".conv"] = torch.zeros_like(w[p + leaf + ".conv"])
                w[p + leaf + ".conv"][:, -1] = 1.0
        w[p + "rel"] = w[p + "rel"] * 0.2
        if i + 1 < len(layers):
            w[p + "o"] = torch.zeros_like(w[p + "o"])
    return Case(tmp, cfg, weights=w), cfg


def asking(window, reach=60, **m):
    return {"type": "attention", "mlp": None, "mixer": dict({"heads": 2, "kv_heads": 1, "dim": 16, "vdim": 32, "conv": 3, "scale": 0.6, "bias_max": reach,
                                                             "mask": {"size": window} if window else None}, **m)}


SHARP = {
    # layers, tokens, places of ASKED with what the last token sees of it
    "window over a page border": ([asking(45)], 301, {300 - 44: True, 300 - 45: False, 299: True, 270: True, 0: False, 3: False}),
    "window in a prompt's middle": ([asking(64, heads=3, dim=10, vdim=9)], 131, {130 - 63: True, 130 - 64: False, 128: True, 129: True}),
    "a window of two": ([asking(2, dim=32, heads=4)], 258, {256: True, 255: False}),
    "a window over three pages": ([asking(300, reach=100)], 560, {559 - 299: True, 559 - 300: False, 511: True, 512: True, 400: True}),
    "everything": ([asking(0, scale=1.0)], 600, {0: True, 3: True, 255: True, 256: True, 257: True, 511: True, 512: True, 598: True}),
    # the second layer reads the first one's keys through a window of its own, wider or narrower than the first one's
    "shared keys, wider window": ([asking(20), shared(asking(50), 0, scale=0.5)], 301, {300 - 49: True, 300 - 50: False, 300 - 20: True, 299: True}),
    "shared keys, narrower window": ([asking(70, dim=10, vdim=12), shared(asking(33, dim=10, vdim=12), 0)], 300, {299 - 32: True, 299 - 33: False, 299 - 69: False}),
}


@pytest.mark.parametrize("name", list(SHARP))
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_key_counts_exactly_where_it_is_seen(tmp_path, dtype, name):
    """The last token asks for one token that lies far back, around page borders, just inside and just outside the window, in its own layer's
    cache and in another's: whole prompt in one step, and the last token decoded alone.  Where the token is seen, the reference's
    logits change with it; where it is not, they do not."""
    layers, n, places = SHARP[name]
    case, cfg = asking_case(tmp_path, layers)
    base = [3 + (i * 7) % 690 for i in range(n - 1)] + [ASKER]
    plain = case.ref(base)[-1:]
    rp = case.replay(dtype, max_tokens=1300)
    try:
        for at, seen in places.items():
            toks = list(base)
            toks[at] = ASKED
            ref = case.ref(toks)[-1:]
            assert (rel_err(ref, plain) > 0.1) if seen else (rel_err(ref, plain) < 1e-9), (at, rel_err(ref, plain))
            whole = rp.step([{"id": 0, "tokens": toks, "want": [n - 1]}], [0])
            rp.step([{"id": 1, "tokens": toks[:n - 1], "want": []}])
            decoded = rp.step([{"id": 1, "tokens": toks[n - 1:], "want": [0]}], [1])
            for got in (whole, decoded):
                assert rel_err(got, ref) < TOL[dtype], at
    finally:
        rp.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_one_distance_stands_out(tmp_path, dtype):
    """A bias table whose rows lie far apart: almost all weight goes to the distances of one bucket, so a bucket edge that is off by one, or a bias
    taken with another head's column, shows; prompts and decoding, with distances beyond the table's reach."""
    cfg = config([asking(70, reach=40, dim=32)], width=64, vocab=90, bias_rows=8)
    w = random_weights(cfg, 14)
    case = Case(tmp_path, cfg, weights=w)
    toks = tokens_of(cfg, 90, 4)
    plain = case.ref(toks)
    rel = torch.zeros(8, 2)
    rp = None
    for b in (0, 3, 4, 5, 6, 7):
        rel = torch.zeros(8, 2)
        rel[b, 0], rel[(b + 3) % 8, 1] = 9.0, 9.0
        w["l0.mix.rel"] = rel.to(torch.bfloat16)
        one = Case(tmp_path / str(b), cfg, weights=w)
        assert rel_err(one.ref(toks), plain) > 0.2
        rp = one.replay(dtype)
        try:
            run_schedule(rp, one, {"a": toks}, [[("a", 71)], [("a", 2)]] + [[("a", 1)]] * 17, dtype)
        finally:
            rp.close()


def test_every_mechanism_shows(tmp_path):
    """With a mechanism taken out of the oracle its logits change clearly, so the agreement of the other tests is not one that the fault
    could share."""
    cfg = config([ATT_A, shared(ATT_A, 0)], width=48, vocab=90)
    case = Case(tmp_path, cfg, seed=4)
    toks = tokens_of(cfg, 60, 1)
    full = case.ref(toks)
    for name in ("bigram", "pos", "l0.mix.rel", "l1.mix.rel", "l0.mix.g", "l1.mix.q.conv", "l0.mlp.shared.up", "l0.norm1.b", "l1.norm2.b", "final.norm.b", "l1.hc1.mix", "l0.hc2.out"):
        W = {k: torch.zeros_like(v) if k == name else v for k, v in case.W.items()}
        assert rel_err(R.forward(W, cfg, toks).numpy(), full) > 20 * TOL["float32"], name
    for name in ("l0.mix.q.conv", "l0.mix.k.conv", "l0.mix.v.conv"):                  # (only the earlier taps)
        W = dict(case.W)
        W[name] = W[name].clone()
        W[name][:, :-1] = 0
        assert rel_err(R.forward(W, cfg, toks).numpy(), full) > 20 * TOL["float32"], name
    W = {k: v.t().contiguous() if k == "l0.hc1.mix" else v for k, v in case.W.items()}       # (from and to exchanged)
    assert rel_err(R.forward(W, cfg, toks).numpy(), full) > 20 * TOL["float32"]
    W = {k: -v if k == "l1.mlp.correction" else v for k, v in case.W.items()}
    assert rel_err(R.forward(W, cfg, toks).numpy(), full) > 20 * TOL["float32"]
    for field, value in (("mask", {"size": 42}), ("bias_max", 24), ("scale", 0.21)):
        other = copy.deepcopy(cfg)
        other["layers"][1]["mixer"][field] = value
        assert rel_err(R.forward(case.W, other, toks).numpy(), full) > 20 * TOL["float32"], field


# ----------------------------------------------------------------------------------------------------- other sizes
def test_sizes_no_kernel_tile_divides(tmp_path):
    """A width that is no multiple of 8; one head; twenty query heads over one key head; a window of one token, and one longer than the sequence;
    no window; one tap, nine taps; one expert; as many choices as experts; no shared expert; one bias row pair; five streams; tensors of
    a feed-forward that the layer does not have."""
    layers = [{"type": "attention", "mlp": {"kind": "moe", "expert": {"ff": 7}, "router": {"experts": 1, "top": 1}, "shared": {"ff": 3}},
               "mixer": {"heads": 1, "kv_heads": 1, "dim": 4, "vdim": 3, "conv": 9, "scale": 0.5, "bias_max": 4, "mask": {"size": 1}}},
              {"type": "attention", "mlp": {"kind": "moe", "expert": {"ff": 5}, "router": {"experts": 3, "top": 3}, "shared": None},
               "mixer": {"heads": 20, "kv_heads": 1, "dim": 4, "vdim": 6, "conv": 1, "scale": 0.5, "bias_max": 3000, "mask": {"size": 5000}}},
              {"type": "attention", "mlp": None,
               "mixer": {"heads": 2, "kv_heads": 1, "dim": 50, "vdim": 30, "conv": 2, "scale": 0.1, "bias_max": 9, "mask": None}},
              {"type": "attention", "mlp": None,
               "mixer": {"heads": 4, "kv_heads": 1, "dim": 50, "vdim": 30, "conv": 3, "scale": 0.2, "bias_max": 60, "mask": {"size": 50}, "kv_from": 2}},
              {"type": "attention", "mlp": {"kind": "moe", "expert": {"ff": 64}, "router": {"experts": 9, "top": 4}, "shared": {"ff": 64}},
               "mixer": {"heads": 3, "kv_heads": 3, "dim": 16, "vdim": 2, "conv": 6, "scale": 0.4, "bias_max": 5, "mask": {"size": 7}}}]
    cfg = config(layers, width=50, vocab=37, streams=5, bias_rows=4, buckets=3)
    cfg["max_positions"] = 80
    for dtype in ("float32", "bfloat16"):
        w = random_weights(cfg, 6, calm=dtype == "bfloat16")
        w["l2.norm2"], w["l2.norm2.b"], w["l3.hc2.mix"] = torch.ones(50).bfloat16(), torch.zeros(50).bfloat16(), torch.eye(5).bfloat16()
        case = Case(tmp_path / dtype, cfg, weights=w)
        toks = tokens_of(cfg, 80, 3)
        rp = case.replay(dtype)
        try:
            run_schedule(rp, case, {"a": toks, "b": toks[:7]}, [[("a", 33), ("b", 5)], [("a", 1), ("b", 2)], [("a", 44)], [("a", 1)], [("a", 1)]], dtype,
                         tol=None if dtype == "float32" else 0.2)      # (50 columns wide: the rounding of bf16 adds up layer by layer)
        finally:
            rp.close()


def test_configs_that_do_not_fit_are_refused():
    from types import SimpleNamespace
    from nanovllm.models.tabedra import TabedraForCausalLM
    make = lambda layers: TabedraForCausalLM(SimpleNamespace(**config(layers, width=32, vocab=20)))
    with pytest.raises(ValueError):
        make([dict(ATT_A, type="unknown")])
    with pytest.raises(ValueError):
        make([dict(ATT_A, mlp={"kind": "dense", "ff": 8})])
    with pytest.raises(ValueError):                                    # keys of a layer that runs later
        make([shared(ATT_A, 1), ATT_A])
    with pytest.raises(AssertionError):                                # keys of other sizes
        make([ATT_A, shared(ATT_B, 0)])
    with pytest.raises(AssertionError):                                # keys of a layer that has none of its own
        make([ATT_A, shared(ATT_A, 0), shared(ATT_A, 1)])
    with pytest.raises(KeyError):
        make([ATT_A]).weight_target("l0.mlp.e6.up")


# ----------------------------------------------------------------------------------------------------- the engine's own entry point
def test_greedy_generation_through_the_engine(mix_case):
    """LLM.generate with temperature 0 (scheduler, chunked prefill, steps launched ahead of their ids, captured graphs, sampling kernel) against
    greedy decoding of the reference."""
    from nanovllm import LLM, SamplingParams
    case = mix_case()
    prompts = [tokens_of(CFG_MIX, n, 50 + n) for n in (5, 40, 17)]
    llm = LLM(case.path, dtype="float32", max_num_seqs=4, max_num_batched_tokens=32, max_model_len=128, num_kvcache_blocks=6, chunked_prefill=True)
    try:
        assert llm.model_runner.graphs, "one-token steps are expected to replay captured graphs"
        outs = llm.generate(prompts, SamplingParams(temperature=0.0, max_tokens=12, ignore_eos=True), use_tqdm=False)
    finally:
        llm.exit()
    for prompt, out in zip(prompts, outs):
        toks = list(prompt)
        for _ in range(12):
            toks.append(int(R.forward(case.W, CFG_MIX, toks)[-1].argmax()))
        assert out["token_ids"] == toks[len(prompt):]


def test_captured_decode_steps_match_eager_ones(flat_case):
    """One-token steps replayed from the captured graph (convolution inputs and last tokens brought up to date in it) against the same steps
    run eagerly: several replays, with eager work between them."""
    from nanovllm.config import Config
    from nanovllm.engine.model_runner import ModelRunner
    from nanovllm.engine.sequence import Sequence
    toks = [tokens_of(CFG_FLAT, n, 70 + n) for n in (60, 11, 47)]
    logits = {}
    for eager in (True, False):
        cfg = Config(flat_case.path, max_num_batched_tokens=128, max_num_seqs=4, max_model_len=128, num_kvcache_blocks=6,
                     chunked_prefill=True, enforce_eager=eager, async_scheduling=False, dtype="float32")
        runner = ModelRunner(cfg, 0, [])
        try:
            seqs = []
            for i, t in enumerate(toks):
                s = Sequence(list(t[:-8]))
                s.block_table, s.num_new_tokens, s.state_slot = [i], len(t) - 8, 3 - i
                seqs.append(s)
            runner.forward_logits(seqs)
            rows = []
            for step in range(8):
                for s, t in zip(seqs, toks):
                    s.num_cached_tokens += s.num_new_tokens
                    s.append_token(t[len(t) - 8 + step])
                    s.num_new_tokens = 1
                out, _, _ = runner.forward_logits(seqs)
                rows.append(out.float().cpu().numpy())
            logits[eager] = np.stack(rows)
            assert eager or runner.graphs
        finally:
            runner.exit()
    assert np.abs(logits[True] - logits[False]).max() < 1e-4 * np.abs(logits[True]).max()
    for i, t in enumerate(toks):
        want = flat_case.ref(t)
        for step in range(8):
            assert rel_err(logits[False][step, i:i + 1], want[len(t) - 8 + step:len(t) - 7 + step]) < TOL["float32"]


def test_the_replay_program_steps_through_a_schedule(tmp_path, mix_case):
    """bin/trace_run as a user starts it: steps on standard input, `done <n>` after each, logits of the wanted places in <out>/<n>.f32;
    a request that is left out of a step and goes on later, one that ends and whose pages and slot the next one takes over."""
    import subprocess
    import sys
    from conftest import ROOT
    a, b = tokens_of(CFG_MIX, 40, 91), tokens_of(CFG_MIX, 12, 92)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:25], "want": [0, 24]}], "end": []},
             {"step": 1, "entries": [{"id": "b", "tokens": b[:10], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": a[25:39], "want": [13]}, {"id": "b", "tokens": b[10:], "want": [1]}], "end": ["b"]},
             {"step": 3, "entries": [{"id": "a", "tokens": a[39:], "want": [0]}], "end": ["a"]}]
    for dtype in ("bfloat16", "float32"):
        case = mix_case(dtype)
        out = tmp_path / dtype
        done = subprocess.run([sys.executable, str(ROOT / "bin" / "trace_run"), "--model", case.path, "--dtype", dtype, "--out", str(out), "--max-tokens", "128"],
                              input="".join(json.dumps(st) + "\n" for st in steps), capture_output=True, text=True, timeout=600)
        assert done.returncode == 0, done.stderr[-2000:]
        assert [ln for ln in done.stdout.splitlines() if ln.startswith("done")] == [f"done {n}" for n in range(4)]
        assert not (out / "1.f32").exists()
        ra, rb = case.ref(a), case.ref(b)
        want = {0: ra[[0, 24]], 2: np.concatenate([ra[38:39], rb[11:12]]), 3: ra[39:40]}
        for n, w in want.items():
            got = np.fromfile(out / f"{n}.f32", dtype="<f4").reshape(-1, CFG_MIX["vocab"])
            assert got.shape == w.shape and rel_err(got, w) < TOL[dtype], (dtype, n)


def test_the_sample_config_is_served_with_random_weights():
    """model_configs/tabedra-1k (layer sizes of a real model; no checkpoint, so the engine draws weights): prompts of unequal
    length are prefilled in chunks and decoded from captured graphs."""
    from conftest import ROOT
    from nanovllm import LLM, SamplingParams
    llm = LLM(str(ROOT / "nano-vllm-v1_amd" / "model_configs" / "tabedra-1k"), max_num_seqs=4, max_num_batched_tokens=256, max_model_len=1024,
              num_kvcache_blocks=12, chunked_prefill=True)
    try:
        prompts = [torch.randint(0, 32768, (n,), generator=torch.Generator().manual_seed(n)).tolist() for n in (600, 3, 130)]
        outs = llm.generate(prompts, SamplingParams(temperature=0.0, max_tokens=8, ignore_eos=True), use_tqdm=False)
        again = llm.generate(prompts[1:2], SamplingParams(temperature=0.0, max_tokens=8, ignore_eos=True), use_tqdm=False)
    finally:
        llm.exit()
    assert all(len(o["token_ids"]) == 8 for o in outs) and again[0]["token_ids"] == outs[1]["token_ids"]
