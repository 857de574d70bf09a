"""Mopalorn through the engine against the plain float64 restatement in tests/mopalorn_reference.py.

Every test makes its own small configuration and random weights (written as config.json + model.safetensors into a
temporary directory, so the config reader and the loader are part of what is tested), runs a schedule through
nanovllm.trace_replay.TraceReplay (the engine's runner, page manager and kernels) and compares logits - and, for
single layers, the residual stream - with the reference run over each whole sequence.  fp32 serving is compared
tightly, bf16 serving within the rounding of its products.
"""
import copy
import json
import math
import os

import numpy as np
import pytest
import torch

import mopalorn_reference as R

pytestmark = pytest.mark.gpu

FF_A, FF_B = {"kind": "dense", "ff": 120}, {"kind": "dense", "ff": 50}
# sizes of the matrix-core attention in bf16 (multiples of 16), window edges inside the test lengths
LAT_A = {"type": "latent_attention", "mlp": FF_A,
         "mixer": {"heads": 3, "dim": 32, "rot_dim": 16, "vdim": 48, "kv_rank": 64, "scale": 0.2, "rot": {"base": 500.0, "dims": 16}, "mask": {"size": 23}}}
# sizes that no tile divides (the vector-ALU attention in both types), no feed-forward
LAT_B = {"type": "latent_attention", "mlp": None,
         "mixer": {"heads": 2, "dim": 10, "rot_dim": 6, "vdim": 14, "kv_rank": 27, "scale": 0.3, "rot": {"base": 90.0, "dims": 6}, "mask": {"size": 41}}}
ATT_A = {"type": "attention", "mlp": FF_A,
         "mixer": {"heads": 4, "kv_heads": 2, "dim": 32, "vdim": 16, "scale": 0.3, "softcap": 4.0, "q_temp": {"coef": 0.7, "every": 10}, "v_mix": True}}
ATT_B = {"type": "attention", "mlp": FF_B,
         "mixer": {"heads": 6, "kv_heads": 2, "dim": 20, "vdim": 12, "scale": 0.25, "softcap": 9.0, "q_temp": {"coef": 0.3, "every": 1}, "v_mix": False}}
POOL_A = {"type": "attention_2", "mlp": FF_B,
          "mixer": {"heads": 4, "kv_heads": 2, "dim": 32, "vdim": 16, "scale": 0.3, "mask": {"size": 20, "pool": 4}, "v_mix": True}}
# blocks of 7: no power of two, so a block lies across a page border; a group of three heads per key head
POOL_B = {"type": "attention_2", "mlp": None,
          "mixer": {"heads": 6, "kv_heads": 2, "dim": 16, "vdim": 16, "scale": 0.4, "mask": {"size": 33, "pool": 7}, "v_mix": True}}
POOL_C = {"type": "attention_2", "mlp": FF_A,
          "mixer": {"heads": 3, "kv_heads": 3, "dim": 12, "vdim": 20, "scale": 0.5, "mask": {"size": 9, "pool": 5}}}


def config(layers, width=96, vocab=131, scale=0.3, eps=1e-5):
    return {"architecture": "Mopalorn", "vocab": vocab, "width": width, "norm": {"eps": eps}, "logit_scale": scale, "layers": copy.deepcopy(layers)}


CFG_MIX = config([LAT_A, POOL_A, LAT_B, ATT_A, POOL_A])                      # the first layer that mixes values is a pooled one
CFG_FLAT = config([ATT_A, POOL_B, LAT_A, POOL_C], width=128, vocab=200, scale=0.8, eps=1e-6)


def random_weights(cfg: dict, seed: int) -> dict:
    """bf16 weights in checkpoint naming."""
    g = torch.Generator().manual_seed(seed)
    D, V = cfg["width"], cfg["vocab"]
    W = {}

    def mat(name, out, inp, scale=1.0):
        W[name] = torch.randn(out, inp, generator=g) * (scale / math.sqrt(inp))

    def vec(name, n, scale=0.2, shift=1.0):
        W[name] = shift + scale * torch.randn(n, generator=g)

    W["embed"] = torch.randn(V, D, generator=g)
    vec("final.norm", D)
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        for n in ("norm1", "norm1b") + (("norm2", "norm2b") if L.get("mlp") else ()):
            vec(p + n, D)
        h, d, dv = m["heads"], m["dim"], m["vdim"]
        if L["type"] == "latent_attention":
            r, n = m["rot_dim"], m["kv_rank"]
            mat(p + "mix.q", h * (d + r), D)
            mat(p + "mix.dkv", n + r, D)
            vec(p + "mix.dkv.norm", n)
            mat(p + "mix.uk", h * d, n)
            mat(p + "mix.uv", h * dv, n)
            mat(p + "mix.g", h * dv, D)
        else:
            kv = m["kv_heads"]
            mat(p + "mix.q", h * d, D)
            mat(p + "mix.k", kv * d, D)
            mat(p + "mix.v", kv * dv, D)
            if L["type"] == "attention_2":
                vec(p + "mix.sink", h, 1.0, 0.5)
            if m.get("v_mix"):
                W[p + "mix.vmix"] = 0.4 + 0.2 * torch.randn((), generator=g)
        mat(p + "mix.o", D, h * dv)
        if L.get("mlp"):
            mat(p + "mlp.up", L["mlp"]["ff"], D, 1.5)
            mat(p + "mlp.down", D, L["mlp"]["ff"])
            W[p + "mlp.act"] = torch.tensor([0.3, -0.6]) + 0.3 * torch.randn(2, generator=g)
    return {k: v.to(torch.bfloat16) for k, v in W.items()}


def write_model(path, cfg: dict, weights: dict) -> str:
    from safetensors.torch import save_file
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file({k: v.contiguous() for k, v in weights.items()}, os.path.join(path, "model.safetensors"))
    return str(path)


class Case:
    """A model on disk, its reference weights and cached reference logits per token list."""

    def __init__(self, tmp, cfg, seed=0, weights=None):
        self.cfg = cfg
        w = weights if weights is not None else random_weights(cfg, seed)
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


TOL = {"float32": 1e-4, "bfloat16": 6e-2}


@pytest.fixture(scope="module")
def mix_case(tmp_path_factory):
    return Case(tmp_path_factory.mktemp("mopalorn_mix"), CFG_MIX, seed=1)


@pytest.fixture(scope="module")
def flat_case(tmp_path_factory):
    return Case(tmp_path_factory.mktemp("mopalorn_flat"), CFG_FLAT, seed=2)


def run_schedule(rp, case, requests: dict, schedule: list, dtype: str, tol=None):
    """schedule: list of steps, each a list of (request id, token count); every position's logits are asked for and
    compared with the reference of the whole request.  Requests end when their tokens are used up."""
    at = {r: 0 for r in requests}
    worst = 0.0
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
            want = case.ref(requests[rid])[lo:hi]
            err = rel_err(got[row:row + hi - lo], want)
            assert err < (tol or TOL[dtype]), f"request {rid} tokens {lo}..{hi}: error {err:.3g}"
            worst = max(worst, err)
            row += hi - lo
    assert all(at[r] == len(requests[r]) for r in requests)
    return worst


# ----------------------------------------------------------------------------------------------------- single mechanisms
@pytest.mark.parametrize("layer", [LAT_A, LAT_B, ATT_A, ATT_B, POOL_A, POOL_B, POOL_C],
                         ids=["latent(matrix cores in bf16)", "latent(ragged, no feed-forward)", "softcap(matrix cores in bf16)", "softcap(ragged, temperature at every position)",
                              "pooled(matrix cores in bf16)", "pooled(blocks of 7, no feed-forward)", "pooled(ragged)"])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_one_layer_stream_matches(tmp_path, layer, dtype):
    """One layer of each kind: the residual stream after it and the logits; 80 tokens cross every window and several blocks."""
    cfg = config([layer], width=72, vocab=50)
    case = Case(tmp_path, cfg, seed=3)
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
    toks = tokens_of(CFG_MIX, 70, 7)
    rp = mix_case.replay("float32")
    try:
        rp.runner.model.collect = []
        rp.step([{"id": 0, "tokens": toks, "want": [0]}], [0])
        streams = [c.cpu().numpy() for c in rp.runner.model.collect]
    finally:
        rp.close()
    col = []
    R.forward(mix_case.W, CFG_MIX, toks, col)
    assert len(streams) == len(col) == 5
    for n, (a, b) in enumerate(zip(streams, col)):
        assert np.abs(a - b.numpy()).max() < 1e-4 * max(1.0, float(b.abs().max())), f"layer {n}"


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


@pytest.mark.parametrize("H,G,d,dv,window,pool", [(4, 2, 32, 32, 40, 8), (4, 2, 32, 16, 20, 7), (6, 2, 20, 12, 33, 5), (2, 2, 64, 64, 1, 1), (8, 1, 16, 32, 300, 64),
                                                  (3, 3, 16, 16, 2, 300), (2, 1, 128, 128, 64, 16), (40, 2, 16, 16, 50, 3)])
def test_pooled_attention_against_dense_softmax(H, G, d, dv, window, pool):
    """The block means written step by step (portions that end inside blocks; one-token steps), then the paged attention over them with a
    window and sinks: prompts, one-query steps (where, in bf16, a group's heads share a workgroup and the tiles - of means and of
    tokens - go to several); sizes for the matrix-core and for the vector-ALU kernel; blocks that lie across pages, of one token, and
    longer than a page."""
    from nanovllm import ops
    g = torch.Generator().manual_seed(6)
    page, rows = 256, -(-256 // pool)
    for cast, tol in ((torch.float32, 1e-4), (torch.bfloat16, 2e-2)):
        lens = [620, 70]
        pages = [[4, 0, 2], [1, 0, 0]]
        q, k, v = ([torch.randn(n, hh, dd, generator=g).to(cast) for n in lens] for hh, dd in ((H, d), (G, d), (G, dv)))
        sinks = torch.randn(H, generator=g) * 2 + 2
        kc, vc = (sum(paged(x[b], pages[b], page, tr) for b in range(2)).cuda() for x, tr in ((k, False), (v, True)))
        tables = torch.tensor(pages, dtype=torch.int32).cuda()
        pk = torch.full((8, rows, G, d), float("nan"), dtype=cast).cuda()            # (nothing but written means may be read)
        pv = torch.full((8, rows, G, dv), float("nan"), dtype=cast).cuda()
        at = [0, 0]
        for take in ([3, 1], [250, 30], [9, 39]):                                    # portions; then single tokens up to the first sequence's end
            at = [at[b] + take[b] for b in range(2)]
            cu = torch.tensor([0, take[0], sum(take)], dtype=torch.int32).cuda()
            ops.attn_pool_blocks(kc, vc, cu, torch.tensor(at, dtype=torch.int32).cuda(), tables, sum(take), pool, pk, pv)
        while at[0] < 300:
            at[0] += 1
            ops.attn_pool_blocks(kc, vc, None, torch.tensor([at[0], 0], dtype=torch.int32).cuda(), tables, 2, pool, pk, pv)      # (the second row is padding)
        cu = torch.tensor([0, 320], dtype=torch.int32).cuda()
        ops.attn_pool_blocks(kc, vc, cu, torch.tensor([620], dtype=torch.int32).cuda(), tables[:1], 320, pool, pk, pv)
        written = 0
        for b in range(2):
            for n in range(lens[b] // pool):
                last = n * pool + pool - 1
                row = n - (last // page * page) // pool
                for x, got in ((k, pk), (v, pv)):
                    mean = x[b][n * pool:last + 1].double().mean(0)
                    assert (got[pages[b][last // page], row].cpu().double() - mean).abs().max() < (1e-5 if cast == torch.float32 else 1e-2), (b, n)
                written += 1
        assert int((~torch.isnan(pk[:, :, 0, 0])).sum()) == written
        for take in ((40, 70), (1, 1), (130, 2)):
            ends = [lens[0] - (5 if take[0] == 1 else 0), lens[1] - (9 if take[1] == 1 else 0)]
            qs = torch.cat([q[b][ends[b] - take[b]:ends[b]] for b in range(2)]).reshape(-1, H * d).cuda()
            cu = torch.tensor([0, take[0], take[0] + take[1]], dtype=torch.int32).cuda()
            out = ops.attn_paged_any(qs, kc, vc, cu if take[0] > 1 else None, torch.tensor(ends, dtype=torch.int32).cuda(), tables, 0.3, H, G, d, dv,
                                     window=window, sinks=sinks.cuda(), pool=pool, pooled=(pk, pv)).cpu().double().view(-1, H, dv)
            row = 0
            for b in range(2):
                for i in range(ends[b] - take[b], ends[b]):
                    if i % 13 == 3 or i >= ends[b] - 2:                               # (a sample of the rows keeps the oracle quick)
                        ref = one_row(q[b][i].double(), k[b].double(), v[b].double(), i, 0.3, window, pool, sinks.double())
                        assert (out[row] - ref).abs().max() < tol * max(1.0, float(ref.abs().max())), (cast, take, b, i)
                    row += 1


def one_row(q, k, v, i, scale, window, pool, sinks):
    """What R.attend gives for position i alone: q [H, d], k [T, G, d], v [T, G, dv]."""
    H, G = q.shape[0], k.shape[1]
    n, first = R.pooled_blocks(i, window, pool), max(0, i - window + 1)
    out = []
    for h in range(H):
        g = h // (H // G)
        keys, vals = (torch.cat([R.block_mean(x[:, g], b, pool)[None] for b in range(n)] + [x[first:i + 1, g]]) for x in (k, v))
        out.append(R.softmax_mix((keys @ q[h]) * scale, vals, sinks[h]))
    return torch.stack(out)


def test_softcap_and_query_temperature_against_dense_softmax():
    """Scores far beyond the cap and far below it, of both signs; a temperature that steps at its multiples."""
    from nanovllm import ops
    g = torch.Generator().manual_seed(8)
    for H, G, d, dv, cap, temp in [(4, 2, 32, 16, 3.0, (0.7, 16)), (6, 2, 20, 12, 15.0, (0.2, 1)), (2, 2, 64, 64, 0.0, (1.5, 100)), (8, 1, 16, 32, 1.0, None),
                                  (2, 2, 48, 48, 0.0, None), (3, 1, 80, 80, 0.0, None), (4, 1, 240, 208, 0.0, None), (5, 1, 112, 96, 20.0, (0.1, 7)), (2, 1, 256, 192, 0.0, None)]:
        for cast, tol in ((torch.float32, 1e-4), (torch.bfloat16, 2e-2)):
            n = 300
            q, k, v = (torch.randn(n, hh, dd, generator=g).to(cast) for hh, dd in ((H, d), (G, d), (G, dv)))
            q = (q.float() * torch.linspace(0.01, 4.0, n)[torch.randperm(n, generator=g)][:, None, None]).to(cast)
            kc, vc = paged(k, [5, 3], 256, False).cuda(), paged(v, [5, 3], 256, True).cuda()
            table = torch.tensor([[5, 3]], dtype=torch.int32).cuda()
            want = R.attend(q.double(), k.double(), v.double(), 0.5, cap=cap, q_temp=None if temp is None else {"coef": temp[0], "every": temp[1]})
            for take, end in ((n, n), (1, n), (1, 1), (50, 260), (1, 16), (1, 15)):
                cu = torch.tensor([0, take], dtype=torch.int32).cuda()
                out = ops.attn_paged_any(q[end - take:end].reshape(take, -1).cuda(), kc, vc, cu if take > 1 else None, torch.tensor([end], dtype=torch.int32).cuda(), table,
                                         0.5, H, G, d, dv, softcap=cap, q_temp=temp).cpu().double().view(take, H, dv)
                assert (out - want[end - take:end]).abs().max() < tol * max(1.0, float(want.abs().max())), (H, d, cap, temp, cast, take, end)


def test_xielu_against_its_formula():
    from nanovllm import ops
    g = torch.Generator().manual_seed(2)
    for rows, inter in [(5, 37), (64, 256), (3, 8)]:
        x = torch.randn(rows, inter + 8, generator=g) * 3
        x[0, :8] = torch.tensor([0.0, -0.0, 1e-4, -1e-4, -30.0, 30.0, -1e-2, 12.0])
        for cast in (torch.float32, torch.bfloat16):
            for params in (torch.tensor([0.4, -1.2]), torch.tensor([-6.0, 25.0]), torch.zeros(2)):
                xa, pa = x.to(cast), params.to(cast)
                want = R.xielu(xa[:, :inter].double(), pa[0], pa[1])
                got = ops.xielu(xa.cuda()[:, :inter], pa.cuda()).cpu()
                assert got.dtype == cast
                err = (got.double() - want).abs() / want.abs().clamp(min=1.0)
                assert err.max() < (2e-6 if cast == torch.float32 else 5e-3), (rows, inter, cast, params)
                assert torch.equal(ops.xielu(xa[:, :inter].contiguous().cuda(), pa.cuda()).cpu(), got)


def test_latent_rows_and_the_gated_head_product():
    """The prep of a query without a latent of its own (rotated parts into the attention's query rows, latent and rotated key part into
    the cache) and the per-head product with a gate per element, against their formulas."""
    from nanovllm import ops
    g = torch.Generator().manual_seed(5)
    for H, d, r, dv, n in [(3, 32, 16, 48, 64), (2, 10, 6, 14, 27), (1, 5, 2, 3, 8)]:
        T, page = 9, 256
        nq = H * (d + r)
        proj = torch.randn(T, nq + n + r + H * dv, generator=g)
        pos = torch.tensor([0, 1, 2, 255, 256, 7, 30, 31, 600])
        slots = torch.tensor([0, 1, 2, 255, 256, 300, -1, 511, 40], dtype=torch.int32)
        w, freq = torch.rand(n, generator=g) + 0.5, torch.tensor([50.0 ** (-2 * i / r) for i in range(r // 2)])
        kc, vc = torch.zeros(2, page, 1, n + r), torch.zeros(2, 1, n, page)
        qa = torch.zeros(T, H * (n + r))
        kg, vg, qg = kc.cuda(), vc.cuda(), qa.cuda()
        cq, gate = ops.latent_prep(proj.cuda(), nq, n, r, H, None, w.cuda(), 1e-5, pos.cuda(), freq.cuda(), 1.0, False, kg, vg, slots.cuda(), False, qg, d)
        assert cq is None and gate is None
        p = proj.double()
        turn = lambda x, t: R.rotate_halves(torch.cat([x.new_zeros(int(pos[t]), 1, r), x.view(1, 1, r)]), {"dims": r, "base": 50.0})[-1, 0]
        for t in range(T):
            for h in range(H):
                want = turn(p[t, h * (d + r) + d:(h + 1) * (d + r)], t)
                assert (qg.cpu().double()[t, h * (n + r) + n:(h + 1) * (n + r)] - want).abs().max() < 2e-4, (t, h)
            s = int(slots[t])
            if s >= 0:
                c = R.rms_norm(p[t, nq:nq + n], w.double(), 1e-5)
                row = kg.cpu().double()[s // page, s % page, 0]
                assert (row[:n] - c).abs().max() < 1e-5 and (row[n:] - turn(p[t, nq + n:nq + n + r], t)).abs().max() < 2e-4
                assert torch.equal(vg.cpu()[s // page, 0, :, s % page], kg.cpu()[s // page, s % page, 0, :n])
        uv, x = torch.randn(H, dv, n, generator=g), torch.randn(T, H * n, generator=g)
        for cast, tol in ((torch.float32, 1e-4), (torch.bfloat16, 0.1)):
            pj, wu, xx = proj.to(cast), uv.to(cast), x.to(cast)
            got = ops.linear_heads(xx.cuda(), wu.cuda(), n, gate=pj.cuda()[:, -H * dv:]).cpu().double()
            want = torch.stack([xx.double().view(T, H, n)[:, h] @ wu[h].double().T for h in range(H)], 1).reshape(T, H * dv) * torch.sigmoid(pj.double()[:, -H * dv:])
            assert (got - want).abs().max() < tol


def test_keys_and_values_go_to_their_slots_with_mixed_values_and_the_means_they_complete():
    """nvh_attn_kv_store: rows that fill several token tiles and columns beyond one column tile, aligned and not, a padded row, with and
    without mixing; then one token per sequence with pooled blocks: the means equal those of nvh_attn_pool_blocks bit for bit."""
    from nanovllm import ops
    g = torch.Generator().manual_seed(9)
    page = 256
    for H, G, d, dv, T in [(4, 2, 12, 10, 5), (4, 2, 32, 16, 37), (3, 3, 64, 96, 20), (2, 1, 5, 150, 17), (1, 1, 3, 1, 1), (2, 1, 10, 16, 515), (1, 1, 72, 64, 640)]:
        proj, first = torch.randn(T, (H + G) * d + G * dv, generator=g), torch.randn(T, 3 + G * dv, generator=g)
        slots = torch.randperm(4 * page, generator=g)[:T].int()
        if T > 2:
            slots[2] = -1
        for cast in (torch.float32, torch.bfloat16):
            for mix in (False, True):
                p, f, lam = proj.to(cast), first.to(cast), torch.tensor([0.37]).to(cast)
                kc, vc = torch.zeros(4, page, G, d, dtype=cast).cuda(), torch.zeros(4, G, dv, page, dtype=cast).cuda()
                pg = p.cuda()
                ops.attn_kv_store(pg[:, H * d:(H + G) * d], pg[:, (H + G) * d:], kc, vc, slots.cuda(), **(dict(v_mix=lam.cuda(), v_first=f.cuda()[:, 3:]) if mix else {}))
                v = p.double()[:, -G * dv:]
                want = (1 - lam.double()) * v + lam.double() * f.double()[:, 3:] if mix else v
                rows_k, rows_v = kc.cpu().view(-1, G * d), vc.cpu().permute(0, 3, 1, 2).reshape(-1, G * dv)
                for t in range(T):
                    s = int(slots[t])
                    if s >= 0:
                        assert torch.equal(rows_k[s], p[t, H * d:(H + G) * d])
                        assert (rows_v[s].double() - want[t]).abs().max() < (1e-6 if cast == torch.float32 else 2e-2)
                assert int((rows_k != 0).any(1).sum()) == int((rows_v != 0).any(1).sum()) == int((slots >= 0).sum())      # nothing else is touched
    for G, d, dv, pool in [(2, 16, 24, 7), (1, 70, 150, 4), (3, 8, 8, 1), (1, 4, 4, 300)]:
        for cast in (torch.float32, torch.bfloat16):
            rows = -(-page // pool)
            kc, vc = torch.randn(6, page, G, d, generator=g).to(cast).cuda(), torch.randn(6, G, dv, page, generator=g).to(cast).cuda()
            tables = torch.tensor([[5, 0], [2, 3], [0, 0], [4, 1]], dtype=torch.int32).cuda()
            for lens in ([7, 300, 0, 256], [259, 8, 0, 4], [256, 301, 0, 266]):
                pos = torch.tensor([max(n - 1, 0) for n in lens])
                slots = torch.tensor([-1 if n == 0 else int(tables[b, (n - 1) // page]) * page + (n - 1) % page for b, n in enumerate(lens)], dtype=torch.int32)
                kv = torch.randn(4, G * (d + dv), generator=g).to(cast).cuda()
                got = [torch.full((6, rows, G, x), 9.0, dtype=cast).cuda() for x in (d, dv)]
                ref = [x.clone() for x in got]
                ops.attn_kv_store(kv[:, :G * d], kv[:, G * d:], kc, vc, slots.cuda(), pool=pool, pooled=tuple(got), positions=pos.cuda(), block_tables=tables)
                ops.attn_pool_blocks(kc, vc, None, torch.tensor(lens, dtype=torch.int32).cuda(), tables, 4, pool, *ref)
                assert torch.equal(got[0], ref[0]) and torch.equal(got[1], ref[1])
                assert int((ref[0] != 9.0).any(-1).any(-1).sum()) == sum(n > 0 and n % pool == 0 for n in lens)


def test_the_one_branch_close_against_its_formula():
    """x + unit(a) w and its norm, four columns a lane (widths around the kernel's pieces) and the general form beside it."""
    from nanovllm import ops
    g = torch.Generator().manual_seed(3)
    for dim in (50, 96, 1024, 1028, 2500, 8192, 8200):
        x, a, wa, wn = torch.randn(5, dim, generator=g) * 3, torch.randn(5, dim, generator=g), torch.randn(dim, generator=g), torch.randn(dim, generator=g)
        for cast in (torch.float32, torch.bfloat16):
            ac, wac, wnc = (t.to(cast) for t in (a, wa, wn))
            for weight in (wac, None):
                branch = R.rms_norm(ac.double(), wac.double(), 1e-5) if weight is not None else ac.double()
                want = x.double() + branch
                xg = x.cuda()
                h = ops.residual_norm(xg, a=ac.cuda(), a_weight=None if weight is None else weight.cuda(), branch_eps=1e-5, norm="rms", weight=wnc.cuda(), eps=1e-3)
                assert (xg.cpu().double() - want).abs().max() < 2e-5
                assert (h.cpu().double() - R.rms_norm(want, wnc.double(), 1e-3)).abs().max() < (2e-5 if cast == torch.float32 else 0.04), (dim, cast)
                xg = x.cuda()
                assert ops.residual_norm(xg, a=ac.cuda(), a_weight=None if weight is None else weight.cuda(), branch_eps=1e-5) is None
                assert (xg.cpu().double() - want).abs().max() < 2e-5


# ----------------------------------------------------------------------------------------------------- schedules
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_prefill_then_token_by_token(mix_case, dtype):
    toks = tokens_of(CFG_MIX, 120, 11)
    rp = mix_case.replay(dtype)
    try:
        run_schedule(rp, mix_case, {"a": toks}, [[("a", 45)]] + [[("a", 1)]] * 75, dtype)
        # the first tokens of a sequence, one by one from the very start (one key, no block yet)
        run_schedule(rp, mix_case, {"b": toks[:40]}, [[("b", 1)]] * 40, dtype)
    finally:
        rp.close()


def test_portions_of_every_size_give_the_same_logits(mix_case):
    toks = tokens_of(CFG_MIX, 120, 13)
    rp = mix_case.replay("float32")
    try:
        for sizes in ([120], [2] * 60, [3, 2, 17, 2, 33, 16, 2, 45], [64, 56], [1, 119], [22, 1, 1, 17, 2, 77]):
            assert sum(sizes) == 120
            run_schedule(rp, mix_case, {"a": toks}, [[("a", s)] for s in sizes], "float32")
    finally:
        rp.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_mixed_batches_of_unequal_requests(mix_case, dtype):
    reqs = {"a": tokens_of(CFG_MIX, 75, 21), "b": tokens_of(CFG_MIX, 9, 22), "c": tokens_of(CFG_MIX, 33, 23), "d": tokens_of(CFG_MIX, 2, 24)}
    sched = [[("a", 30), ("b", 3)], [("a", 1), ("b", 2), ("c", 20)], [("b", 1), ("a", 17), ("c", 1), ("d", 2)], [("c", 2), ("a", 27), ("b", 3)],
             [("c", 10)]]
    rp = mix_case.replay(dtype)
    try:
        run_schedule(rp, mix_case, reqs, sched, dtype)
    finally:
        rp.close()


def test_pages_are_used_again(flat_case):
    """A pool of three pages serves six requests one after another and in pairs: every request after the first two runs on pages
    (keys, values, block means) that others have left behind."""
    reqs = {i: tokens_of(CFG_FLAT, n, 30 + i) for i, n in enumerate([300, 120, 257, 40, 256, 130])}
    rp = flat_case.replay("float32", max_tokens=256, slots=2)            # ceil(256/256) + 2 = 3 pages
    assert len(rp.scheduler.block_manager.blocks) == 3
    try:
        run_schedule(rp, flat_case, {0: reqs[0]}, [[(0, 200)], [(0, 100)]], "float32")
        run_schedule(rp, flat_case, {1: reqs[1], 2: reqs[2]}, [[(1, 100), (2, 7)], [(1, 20), (2, 250)]], "float32")
        run_schedule(rp, flat_case, {3: reqs[3], 4: reqs[4]}, [[(4, 255), (3, 39)], [(3, 1), (4, 1)]], "float32")
        run_schedule(rp, flat_case, {5: reqs[5]}, [[(5, 129)], [(5, 1)]], "float32")
        assert len(rp.scheduler.block_manager.free_block_ids) == 3
        run_schedule(rp, flat_case, {"again": reqs[0]}, [[("again", 300)]], "float32")      # a replayed request is computed anew, no page stands in for it
    finally:
        rp.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_page_borders_in_prompts_and_in_decoding(flat_case, dtype):
    """Portions that end one token before, at and after a page border (a block of seven lies across it), then decoding across the next
    one; portions that end around window and block edges."""
    toks = tokens_of(CFG_FLAT, 530, 41)
    rp = flat_case.replay(dtype, max_tokens=1100)
    try:
        run_schedule(rp, flat_case, {"a": toks}, [[("a", 255)], [("a", 1)], [("a", 1)], [("a", 2)], [("a", 251)], [("a", 3)]] + [[("a", 1)]] * 17, dtype)
        for first in (22, 23, 24, 33, 34, 39, 40, 41, 252, 259, 260):
            run_schedule(rp, flat_case, {"b": toks[:first + 9]}, [[("b", first)], [("b", 7)], [("b", 1)], [("b", 1)]], dtype)
    finally:
        rp.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_one_token_steps_of_sequences_of_unequal_length(flat_case, dtype):
    """Steps in which every sequence brings one token: contexts without and with block means side by side; then fewer sequences as the
    short requests end."""
    reqs = {i: tokens_of(CFG_FLAT, n, 80 + i) for i, n in enumerate([36, 75, 135, 300])}
    first = {0: 30, 1: 64, 2: 129, 3: 290}
    sched = [[(i, first[i]) for i in reqs]] + [[(i, 1) for i in reqs if first[i] + k < len(reqs[i])] for k in range(11)]
    rp = flat_case.replay(dtype, max_tokens=1100)
    try:
        run_schedule(rp, flat_case, reqs, [st for st in sched if st], dtype)
    finally:
        rp.close()


def test_long_decoding(mix_case):
    toks = tokens_of(CFG_MIX, 270, 43)
    rp = mix_case.replay("float32", max_tokens=512)
    try:
        run_schedule(rp, mix_case, {"a": toks}, [[("a", 5)]] + [[("a", 1)]] * 265, "float32")
    finally:
        rp.close()


# ----------------------------------------------------------------------------------------------------- faults that random weights would hide
ASKER, ASKED = 1, 2          # token ids: the query of ASKER scores high on the key of ASKED, all other scores are near zero


def asking_case(tmp, layer, strength, sink=None):
    """One layer whose heads compare one coordinate: only ASKED's key has it, only ASKER's query reads it.  Values are random, so what
    the last token sees of ASKED shows in its logits."""
    cfg = config([layer], width=64, vocab=700)
    w = random_weights(cfg, 9)
    m, p = layer["mixer"], "l0.mix."
    h, d = m["heads"], m["dim"]
    w["embed"][:, :2] = 0
    w["embed"][ASKED, 0] = w["embed"][ASKER, 1] = 8.0
    w["l0.norm1"][:2] = 1.0
    per = d + m.get("rot_dim", 0)
    q = torch.zeros(h, per, 64)
    q[:, 0, 1] = strength
    w[p + "q"] = q.reshape(h * per, 64).to(torch.bfloat16)
    if layer["type"] == "latent_attention":
        n, r = m["kv_rank"], m["rot_dim"]
        w[p + "dkv"][0] = 0
        w[p + "dkv"][0, 0] = 3.0                                           # the latent's first coordinate marks ASKED ...
        w[p + "dkv.norm"][0] = 1.0
        uk = torch.zeros(h, d, n)
        uk[:, 0, 0] = 1.0                                                  # ... and every head's key takes it over
        w[p + "uk"] = uk.reshape(h * d, n).to(torch.bfloat16)
    else:
        k = torch.zeros(m["kv_heads"], d, 64)
        k[:, 0, 0] = 1.0
        w[p + "k"] = k.reshape(-1, 64).to(torch.bfloat16)
        w[p + "v"] = w[p + "v"] * 3
        if sink is not None:
            w[p + "sink"] = torch.tensor(sink).to(torch.bfloat16)
    return Case(tmp, cfg, weights=w), cfg


SHARP = {
    # layer, strength, sinks, tokens, places of ASKED with what the last token sees of it
    "window": ({"type": "latent_attention", "mlp": None,
                "mixer": {"heads": 2, "dim": 16, "rot_dim": 16, "vdim": 32, "kv_rank": 32, "scale": 1.0, "rot": {"base": 300.0, "dims": 16}, "mask": {"size": 45}}}, 2.0, None, 301,
               {300 - 44: True, 300 - 45: False, 299: True, 270: True, 0: False, 3: False}),                   # the window opens on a page border (256)
    "window in a prompt's middle": ({"type": "latent_attention", "mlp": None,
                                     "mixer": {"heads": 3, "dim": 10, "rot_dim": 4, "vdim": 9, "kv_rank": 20, "scale": 1.0, "rot": {"base": 300.0, "dims": 4}, "mask": {"size": 64}}}, 2.0,
                                    None, 131, {130 - 63: True, 130 - 64: False, 128: True}),
    "everything": ({"type": "attention", "mlp": None,
                    "mixer": {"heads": 4, "kv_heads": 2, "dim": 16, "vdim": 32, "scale": 1.0, "softcap": 12.0, "q_temp": {"coef": 0.5, "every": 50}}}, 0.25, None, 600,
                   {0: True, 3: True, 255: True, 256: True, 257: True, 511: True, 512: True, 598: True}),
    # window 40 behind position 330: tokens from 291 on, blocks of 8 up to the one that ends at 287; 288 - 290 are seen by nothing
    "blocks of 8": ({"type": "attention_2", "mlp": None, "mixer": {"heads": 2, "kv_heads": 1, "dim": 16, "vdim": 32, "scale": 1.0, "mask": {"size": 40, "pool": 8}}}, 1.6, [2.0, 4.5], 331,
                    {0: True, 7: True, 255: True, 256: True, 280: True, 287: True, 288: False, 290: False, 291: True, 329: True}),
    # blocks of 12: one of them is 252 - 263, across the page border; window 30 behind 293 opens at 264, right behind it
    "blocks across pages": ({"type": "attention_2", "mlp": None, "mixer": {"heads": 2, "kv_heads": 2, "dim": 20, "vdim": 12, "scale": 1.0, "mask": {"size": 30, "pool": 12}}}, 2.2, [1.0, 3.5], 294,
                            {0: True, 251: True, 252: True, 255: True, 256: True, 263: True, 264: True, 292: True}),
    # ... and behind 292, where the block's last position is still the window's first: its other positions are seen by nothing
    "a block not yet whole": ({"type": "attention_2", "mlp": None, "mixer": {"heads": 2, "kv_heads": 2, "dim": 16, "vdim": 16, "scale": 1.0, "mask": {"size": 30, "pool": 12}}}, 2.2, [1.0, 3.5], 293,
                              {251: True, 252: False, 255: False, 256: False, 262: False, 263: True, 264: True}),
}


@pytest.mark.parametrize("name", list(SHARP))
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_key_counts_exactly_where_it_is_seen(tmp_path, dtype, name):
    """The last token asks for one token that lies far back, around page borders, just inside and just outside the window, in the last
    block that is seen and in the first that is not: whole prompt in one step, and the last token decoded alone.  Where the token is
    seen, the reference's logits change with it; where it is not, they do not."""
    layer, strength, sink, n, places = SHARP[name]
    case, cfg = asking_case(tmp_path, layer, strength, sink)
    base = [3 + (i * 7) % 690 for i in range(n - 1)] + [ASKER]
    plain = case.ref(base)[-1:]
    if sink is not None:
        W = dict(case.W)
        W["l0.mix.sink"] = torch.full_like(W["l0.mix.sink"], -30.0)
        assert rel_err(R.forward(W, cfg, base).numpy()[-1:], plain) > 5e-3         # without the sink the logits are others
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


def test_mixing_temperature_and_sinks_show(tmp_path):
    """With a mechanism taken out of the oracle its logits change clearly, so the agreement of the other tests is not one that the fault
    could share."""
    cfg = config([POOL_A, ATT_A], width=48, vocab=90)
    case = Case(tmp_path, cfg, seed=4)
    toks = tokens_of(cfg, 60, 1)
    full = case.ref(toks)
    for change in ({"l1.mix.vmix": 0.0}, {"l0.mix.sink": -30.0}, {"l0.mlp.act": 0.0}):
        W = {k: torch.full_like(v, change[k]) if k in change else v for k, v in case.W.items()}
        assert rel_err(R.forward(W, cfg, toks).numpy(), full) > 20 * TOL["float32"], change
    assert rel_err(R.forward({k: torch.full_like(v, 9.0) if k == "l0.mix.vmix" else v for k, v in case.W.items()}, cfg, toks).numpy(), full) == 0      # (unused)
    for field, value in (("q_temp", None), ("softcap", 0.0)):
        other = copy.deepcopy(cfg)
        other["layers"][1]["mixer"][field] = value
        assert rel_err(R.forward(case.W, other, toks).numpy(), full) > 20 * TOL["float32"], field
    other = copy.deepcopy(cfg)
    other["layers"][0]["mixer"]["mask"]["pool"] = 1000                     # no block is ever whole
    assert rel_err(R.forward(case.W, other, toks).numpy(), full) > 20 * TOL["float32"]


# ----------------------------------------------------------------------------------------------------- other sizes
def test_sizes_no_kernel_tile_divides(tmp_path):
    """A width that is no multiple of 8; one head; twenty query heads over one key head; windows and blocks of one token, and longer than
    the sequence; a latent wider than the matrix-core kernel takes; a two-wide rotated part; a checkpoint without the unused mixing
    number of the first mixing layer; a layer without value mixing between two that mix."""
    layers = [{"type": "latent_attention", "mlp": {"kind": "dense", "ff": 7},
               "mixer": {"heads": 1, "dim": 4, "rot_dim": 2, "vdim": 3, "kv_rank": 5, "scale": 0.5, "rot": {"base": 50.0, "dims": 2}, "mask": {"size": 1}}},
              {"type": "attention_2", "mlp": None,
               "mixer": {"heads": 20, "kv_heads": 1, "dim": 4, "vdim": 6, "scale": 0.5, "mask": {"size": 1, "pool": 1}, "v_mix": True}},
              {"type": "attention", "mlp": {"kind": "dense", "ff": 33},
               "mixer": {"heads": 2, "kv_heads": 1, "dim": 50, "vdim": 30, "scale": 0.1, "softcap": 2.0, "q_temp": {"coef": 1.0, "every": 1000}, "v_mix": False}},
              {"type": "latent_attention", "mlp": None,
               "mixer": {"heads": 2, "dim": 6, "rot_dim": 10, "vdim": 8, "kv_rank": 290, "scale": 0.3, "rot": {"base": 7.0, "dims": 10}, "mask": {"size": 5000}}},
              {"type": "attention", "mlp": None,
               "mixer": {"heads": 3, "kv_heads": 3, "dim": 16, "vdim": 2, "scale": 0.4, "softcap": 30.0, "q_temp": {"coef": 0.25, "every": 3}, "v_mix": True}},
              {"type": "attention_2", "mlp": {"kind": "dense", "ff": 16},
               "mixer": {"heads": 2, "kv_heads": 2, "dim": 16, "vdim": 3, "scale": 0.4, "mask": {"size": 3000, "pool": 4000}, "v_mix": True}}]
    cfg = config(layers, width=50, vocab=37, scale=1.0)
    w = random_weights(cfg, 6)
    del w["l1.mix.vmix"]
    case = Case(tmp_path, cfg, weights=w)
    toks = tokens_of(cfg, 80, 3)
    for dtype in ("float32", "bfloat16"):
        rp = case.replay(dtype)
        try:
            run_schedule(rp, case, {"a": toks, "b": toks[:7]}, [[("a", 33), ("b", 5)], [("a", 1), ("b", 2)], [("a", 44)], [("a", 1)], [("a", 1)]], dtype,
                         tol=None if dtype == "float32" else 0.15)     # (50 columns wide: the rounding of bf16 adds up layer by layer)
        finally:
            rp.close()
    from types import SimpleNamespace
    from nanovllm.models.mopalorn import MopalornForCausalLM
    with pytest.raises(ValueError):
        MopalornForCausalLM(SimpleNamespace(**config([dict(LAT_B, type="unknown")])))
    with pytest.raises(AssertionError):                                # values of unequal sizes cannot be mixed
        MopalornForCausalLM(SimpleNamespace(**config([ATT_A, dict(POOL_C, mixer=dict(POOL_C["mixer"], v_mix=True))])))


# ----------------------------------------------------------------------------------------------------- the engine's own entry point
def test_greedy_generation_through_the_engine(mix_case):
    """LLM.generate with temperature 0 (scheduler, chunked prefill, captured graphs, sampling kernel) against greedy decoding of
    the reference."""
    from nanovllm import LLM, SamplingParams
    prompts = [tokens_of(CFG_MIX, n, 50 + n) for n in (5, 40, 17)]
    llm = LLM(mix_case.path, dtype="float32", max_num_seqs=4, max_num_batched_tokens=32, max_model_len=128, num_kvcache_blocks=6,
              chunked_prefill=True)
    try:
        assert llm.model_runner.graphs, "one-token steps are expected to replay captured graphs"
        outs = llm.generate(prompts, SamplingParams(temperature=0.0, max_tokens=12, ignore_eos=True), use_tqdm=False)
    finally:
        llm.exit()
    for prompt, out in zip(prompts, outs):
        toks = list(prompt)
        for _ in range(12):
            toks.append(int(R.forward(mix_case.W, CFG_MIX, toks)[-1].argmax()))
        assert out["token_ids"] == toks[len(prompt):]


def test_prompts_with_a_common_prefix_share_its_pages(tmp_path):
    """No layer keeps a state beside its pages, so the engine's prefix cache serves this design: a second prompt that opens with the
    first one's 530 tokens is given their two full pages - keys, values and the block means in them (a block of seven lies across
    each border) - computes the rest, and generates what the reference generates."""
    from nanovllm import LLM, SamplingParams
    cfg = config([POOL_B, ATT_A], width=64, vocab=150)
    case = Case(tmp_path, cfg, seed=12)
    first = tokens_of(cfg, 530, 61)
    second = first + tokens_of(cfg, 25, 62)
    llm = LLM(case.path, dtype="float32", max_num_seqs=2, max_num_batched_tokens=256, max_model_len=800, num_kvcache_blocks=12, chunked_prefill=True)
    try:
        sp = SamplingParams(temperature=0.0, max_tokens=4, ignore_eos=True)
        llm.generate([first], sp, use_tqdm=False)
        from nanovllm.engine.sequence import Sequence
        used, free, new = llm.scheduler.block_manager.get_token_layout(Sequence(list(second)))
        assert used + free == 512 and new == len(second) - 512
        out = llm.generate([second], sp, use_tqdm=False)[0]["token_ids"]
    finally:
        llm.exit()
    toks = list(second)
    for _ in range(4):
        toks.append(int(R.forward(case.W, cfg, toks)[-1].argmax()))
    assert out == toks[len(second):]


def test_captured_decode_steps_match_eager_ones(flat_case):
    """One-token steps replayed from the captured graph (block means included) against the same steps run eagerly: several replays,
    with eager work between them."""
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
                s.block_table, s.num_new_tokens = [i], len(t) - 8
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
    a request that is left out of a step and goes on later, one that ends and whose pages the next one takes over."""
    import subprocess
    import sys
    from conftest import ROOT
    a, b = tokens_of(CFG_MIX, 40, 91), tokens_of(CFG_MIX, 12, 92)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:25], "want": [0, 24]}], "end": []},
             {"step": 1, "entries": [{"id": "b", "tokens": b[:10], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": a[25:39], "want": [13]}, {"id": "b", "tokens": b[10:], "want": [1]}], "end": ["b"]},
             {"step": 3, "entries": [{"id": "a", "tokens": a[39:], "want": [0]}], "end": ["a"]}]
    for dtype in ("bfloat16", "float32"):
        out = tmp_path / dtype
        done = subprocess.run([sys.executable, str(ROOT / "bin" / "trace_run"), "--model", mix_case.path, "--dtype", dtype, "--out", str(out), "--max-tokens", "128"],
                              input="".join(json.dumps(st) + "\n" for st in steps), capture_output=True, text=True, timeout=600)
        assert done.returncode == 0, done.stderr[-2000:]
        assert [ln for ln in done.stdout.splitlines() if ln.startswith("done")] == [f"done {n}" for n in range(4)]
        assert not (out / "1.f32").exists()
        ra, rb = mix_case.ref(a), mix_case.ref(b)
        want = {0: ra[[0, 24]], 2: np.concatenate([ra[38:39], rb[11:12]]), 3: ra[39:40]}
        for n, w in want.items():
            got = np.fromfile(out / f"{n}.f32", dtype="<f4").reshape(-1, CFG_MIX["vocab"])
            assert got.shape == w.shape and rel_err(got, w) < TOL[dtype], (dtype, n)


def test_the_sample_config_is_served_with_random_weights():
    """model_configs/mopalorn-mixed-1k (layer sizes of a real model; no checkpoint, so the engine draws weights): prompts of unequal
    length are prefilled in chunks and decoded from captured graphs."""
    from conftest import ROOT
    from nanovllm import LLM, SamplingParams
    llm = LLM(str(ROOT / "nano-vllm-v1_amd" / "model_configs" / "mopalorn-mixed-1k"), max_num_seqs=4, max_num_batched_tokens=256, max_model_len=1024,
              num_kvcache_blocks=12, chunked_prefill=True)
    try:
        prompts = [torch.randint(0, 32768, (n,), generator=torch.Generator().manual_seed(n)).tolist() for n in (600, 3, 130)]
        outs = llm.generate(prompts, SamplingParams(temperature=0.0, max_tokens=8, ignore_eos=True), use_tqdm=False)
        again = llm.generate(prompts[1:2], SamplingParams(temperature=0.0, max_tokens=8, ignore_eos=True), use_tqdm=False)
    finally:
        llm.exit()
    assert all(len(o["token_ids"]) == 8 for o in outs) and again[0]["token_ids"] == outs[1]["token_ids"]
