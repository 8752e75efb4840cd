"""Revesun (minGRU + chunked attention decoder) against the plain implementation of
oracle_revesun.py: every mechanism alone, then whole models through the engine.

CPU tensors take the framework's PyTorch ops; the ``cuda`` cases run the HIP kernels in f32 (tight)
and bf16 (rounding of bf16 matrix products allowed)."""
import io
import json
import os
import sys

import numpy as np
import pytest
import torch

sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))
import oracle_revesun as orc  # noqa: E402

from mxllm.models import Revesun, RevesunConfig, build_model, model_config, save_revesun  # noqa: E402
from mxllm.ops import hybrid as hops  # noqa: E402
from mxllm.serve.engine import Engine  # noqa: E402
from mxllm.serve.kvcache import KVCache  # noqa: E402

CASES = [("cpu", torch.float32), pytest.param("cuda", torch.float32, marks=pytest.mark.gpu),
         pytest.param("cuda", torch.bfloat16, marks=pytest.mark.gpu)]
on_devices = pytest.mark.parametrize("dev,dt", CASES, ids=lambda x: str(x).replace("torch.", ""))


def close(got, want, dt, scale=1.0):
    """Relative RMS error of the whole, and no element far out."""
    got, want = got.detach().double().cpu(), want.detach().double().cpu()
    tol = (2e-5 if dt == torch.float32 else 1.5e-2) * scale
    rms = want.pow(2).mean().sqrt().clamp_min(1e-6)
    err = (got - want).abs()
    assert torch.isfinite(got).all()
    assert err.pow(2).mean().sqrt() <= tol * rms, (float(err.pow(2).mean().sqrt()), float(rms))
    assert err.max() <= 12 * tol * max(float(rms), float(want.abs().max()) / 4), (float(err.max()), float(rms))


def rnd(*shape, seed=0, dt=torch.float32):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed)).to(dt)


# ------------------------------------------------------------------ mechanisms
@on_devices
@pytest.mark.parametrize("width,groups", [(24, 1), (30, 3), (50, 5), (64, 8), (520, 1), (4608, 1), (4608, 8), (18, 18),
                                          (6000, 1), (3003, 3)])
def test_group_norm(dev, dt, width, groups):
    """Odd part sizes, parts of one element, parts wider than a wave and than a workgroup's registers."""
    x, d = rnd(5, width, seed=1) * torch.linspace(0.01, 3, width), rnd(5, width, seed=2, dt=dt)
    w = 1 + 0.3 * rnd(width, seed=3)
    for delta in (None, d):
        h = x.clone().to(dev)
        y = hops.group_norm(None if delta is None else delta.to(dev), h, w.to(dev), groups, 1e-3, dt)
        res = x if delta is None else x + delta.float()
        assert torch.equal(h.cpu(), res)
        close(y, orc.group_norm(res.double(), w.double(), groups, 1e-3), dt)


@on_devices
@pytest.mark.parametrize("ff", [8, 37, 160, 2048, 5000, 21504])
def test_poly_norm(dev, dt, ff):
    z = (rnd(4, ff, seed=4) * 2 + 0.3).to(dt)
    coef = torch.tensor([0.7, -0.4, 0.3, 0.2])
    y = hops.poly_norm(z.to(dev), coef.to(dev), 1e-5)
    close(y, orc.poly_norm(z.double(), coef.double(), 1e-5), dt)


def scan_inputs(T, W, dt, seed=0):
    x = rnd(T, 3 * W, seed=seed, dt=dt)
    x[:, :W] -= 2.5  # slow gates: a state lost hundreds of tokens back still shows
    return x, 0.5 * rnd(2 * W, seed=seed + 1)


def scan_oracle(x, bias, W, state=None):
    z, u, g = x.double().split(W, 1)
    s = orc.min_gru(z + bias[:W].double(), u + bias[W:].double(), state)
    return s * (g * torch.sigmoid(g)), s[-1]


@on_devices
@pytest.mark.parametrize("W", [5, 96])
def test_min_gru_prompts_and_steps(dev, dt, W):
    """Unequal prompts in one scan (one token, around and far past a scan chunk), end states by slot, then
    single tokens from those states; slots that held another sequence before."""
    lens, slots = [1, 16, 17, 700, 2, 129], [3, 0, 5, 1, 4, 2]
    x, bias = scan_inputs(sum(lens), W, dt)
    state = torch.full((7, W), 9.0, device=dev)  # left over from other sequences
    caches = hops.SeqCaches([], [], None, [], [state])
    y = hops.min_gru(x.to(dev), bias.to(dev), hops.PromptRows(lens, dev, slots, caches), 0)
    at, ends = 0, []
    for n, s in zip(lens, slots):
        want, end = scan_oracle(x[at:at + n], bias, W)
        close(y[at:at + n], want, dt)
        close(state[s], end, torch.float32, 5 if dt == torch.float32 else 50)
        ends.append(end)
        at += n
    assert (state[6] == 9).all()
    x2, _ = scan_inputs(len(lens), W, dt, seed=7)
    rows = hops.TokenRows(torch.tensor(lens, dtype=torch.int32, device=dev),
                          torch.tensor(slots, dtype=torch.int32, device=dev), 1024, caches)
    y2 = hops.min_gru(x2.to(dev), bias.to(dev), rows, 0)
    for i, end in enumerate(ends):
        want, _ = scan_oracle(x2[i:i + 1], bias, W, end)
        close(y2[i:i + 1], want, dt)


def test_scan_chunks_shrink_with_the_work():
    """Narrow scans are cut into chunks of 16 rows, wide ones longer; each covers its rows once."""
    for T, W in ((40, 8), (4096, 4096), (9000, 9000)):
        r = hops.PromptRows([T, 7], "cpu")
        ch, sq, multi = r.scan_tables(W)
        assert multi and int(ch[:, 1].sum()) == T + 7 and int(sq[:, 2].sum()) == len(ch)
        assert int(ch[:, 1].max()) >= 16 and int(ch[:, 3].sum()) == 2


ATTN = [  # heads, kv, dim, vdim, taps, chunk, rot dims
    (4, 2, 16, 16, 4, 24, 8), (2, 2, 20, 12, 3, 7, 20), (6, 1, 32, 48, 2, 37, 2), (4, 4, 64, 64, 4, 130, 64),
    (8, 2, 128, 96, 5, 300, 30), (2, 1, 160, 72, 4, 40, 32), (3, 3, 10, 6, 1, 16, 0), (1, 1, 7, 5, 4, 1, 4),
    (34, 2, 8, 16, 3, 50, 4), (2, 1, 100, 100, 6, 512, 100)]


def attn_setup(case, dt, seed=0):
    H, G, D, E, taps, chunk, rd = case
    sh = hops.AttnShape(H, G, D, E, taps, chunk, rd, 1.7 / D ** 0.5)
    conv = 0.4 * rnd(taps, sh.conv_channels, seed=seed)
    conv[-1] += 1
    return sh, conv


def attn_caches(sh, slots, max_seq, dt, dev):
    kv = KVCache(1, 0, 0, dt, torch.device(dev), slots, max_seq, pool_tokens=slots * 512,
                 shapes=[(sh.kv_heads, *sh.row_dims(dt))], span=sh.chunk)
    ring = torch.full((slots, sh.taps, sh.conv_channels), 5.0, dtype=dt, device=dev)  # a former sequence's values
    return kv, hops.SeqCaches(kv.k, kv.v, kv.bt, [ring], [])


def attn_oracle(x, conv, sh, base=1e4, chunk=None):
    T, C = x.shape[0], sh.conv_channels
    H, G, D, E = sh.heads, sh.kv_heads, sh.dim, sh.vdim
    x = x.double()
    y = orc.causal_conv(x[:, :C], conv.double().T)
    pos = torch.arange(T)
    q = orc.rotate_pairs(y[:, :H * D].view(T, H, D), pos, base, sh.rot_dims)
    k = orc.rotate_pairs(y[:, H * D:(H + G) * D].view(T, G, D), pos, base, sh.rot_dims)
    o = orc.chunk_attention(q, k, y[:, (H + G) * D:].view(T, G, E), sh.scale, chunk or sh.chunk)
    return o.reshape(T, H * E) * torch.sigmoid(x[:, C:])


def tables(sh, n, dev, base=1e4):
    return hops.pair_rope_tables(n, sh.rot_dims, base, device=dev)


@on_devices
@pytest.mark.parametrize("case", ATTN, ids=str)
def test_sink_attention_prompts_and_steps(dev, dt, case):
    """Unequal prompts in one pass, then decoding past several chunk edges, batched; blocks out of order
    and caches that held another sequence."""
    sh, conv = attn_setup(case, dt)
    width = sh.conv_channels + sh.heads * sh.vdim
    lens, slots, more = [1, sh.chunk, 45, 3, max(1, sh.chunk - 1)], [2, 0, 4, 1, 3], 30
    cos, sin = tables(sh, 700, dev)
    kv, caches = attn_caches(sh, 5, 640, dt, dev)
    for s in (4, 2, 0, 3, 1):  # scattered blocks
        kv.reserve(s, 640)
    for c in kv.k + kv.v:
        dims = (slice(None),) * 3 + (slice(0, sh.dim if c is kv.k[0] else sh.vdim),)
        c[dims] = 3.0  # stale rows
    xs = [rnd(n + more, width, seed=10 + i, dt=dt) for i, n in enumerate(lens)]
    want = [attn_oracle(x, conv, sh) for x in xs]
    rows = hops.PromptRows(lens, dev, slots, caches)
    x0 = torch.cat([x[:n] for x, n in zip(xs, lens)]).to(dev)
    y = hops.sink_attention(x0, conv.to(dev), cos, sin, sh, rows, 0)
    close(y, torch.cat([w[:n] for w, n in zip(want, lens)]), dt)
    # without caches the prompt pass is the same
    y2 = hops.sink_attention(x0, conv.to(dev), cos, sin, sh, hops.PromptRows(lens, dev), 0)
    assert torch.equal(y, y2)
    sl = torch.tensor(slots, dtype=torch.int32, device=dev)
    got = []
    for t in range(more):
        pos = torch.tensor([n + t for n in lens], dtype=torch.int32, device=dev)
        xt = torch.stack([x[n + t] for x, n in zip(xs, lens)]).to(dev)
        got.append(hops.sink_attention(xt, conv.to(dev), cos, sin, sh, hops.TokenRows(pos, sl, 640, caches), 0))
    got = torch.stack(got, 1)
    for i, n in enumerate(lens):
        close(got[i], want[i][n:], dt)


@on_devices
@pytest.mark.parametrize("chunk", [20, 128, 300])
def test_chunk_edges_with_a_key_that_stands_out(dev, dt, chunk):
    """One key takes nearly all the weight: the first and last position of a chunk, and the positions just
    outside it.  A mask one position off moves the output by more than a hundred tolerances."""
    sh = hops.AttnShape(2, 1, 32, 32, 2, chunk, 0, 1.0)
    D, C = sh.dim, sh.conv_channels
    T = 2 * chunk + 5
    conv = torch.zeros(2, C)
    conv[1] = 1  # identity
    cos, sin = tables(sh, T + 8, dev)
    for key in (0, 1, chunk - 1, chunk, chunk + 1, 2 * chunk - 1, 2 * chunk):
        x = 0.05 * rnd(T, C + 64, seed=key, dt=dt)
        x[:, :2 * D] = 0
        x[:, 0] = x[:, D] = 4.0           # every query, both heads
        x[key, 2 * D] = 4.0               # the key
        x[key, 3 * D:4 * D] = 1.0         # its value
        want = attn_oracle(x, conv, sh)
        last = min(T, (key // chunk + 1) * chunk)
        # the oracle shows where it is seen
        assert (want[key:last, :].mean(1) > 0.3).all() and (want[:key].mean(1).abs() < 0.2).all()
        assert last == T or (want[last:].mean(1).abs() < 0.2).all()
        wrong = attn_oracle(x, conv, sh, chunk=chunk + 1)
        if 0 < key:
            assert (wrong - want).abs().max() > 0.3
        for n in sorted({1, max(1, key), key + 1, last - 1, last, T - 3}):
            if not 0 < n < T:
                continue
            kv, caches = attn_caches(sh, 1, 640, dt, dev)
            kv.reserve(0, T)
            y = hops.sink_attention(x[:n].to(dev), conv.to(dev), cos, sin, sh, hops.PromptRows([n], dev, [0], caches), 0)
            close(y, want[:n], dt)
            for p in range(n, min(T, n + 4)):
                rows = hops.TokenRows(torch.tensor([p], dtype=torch.int32, device=dev),
                                      torch.zeros(1, dtype=torch.int32, device=dev), 640, caches)
                y = hops.sink_attention(x[p:p + 1].to(dev), conv.to(dev), cos, sin, sh, rows, 0)
                close(y, want[p:p + 1], dt)


@on_devices
def test_softmax_sink(dev, dt):
    """Scores far below 0 leave the weight to the sink, far above 0 take it all."""
    sh = hops.AttnShape(2, 2, 16, 16, 1, 64, 0, 1.0)
    C, T = sh.conv_channels, 9
    cos, sin = tables(sh, T, dev)
    for level in (-30.0, -3.0, 0.0, 6.0, 200.0):
        x = rnd(T, C + 32, seed=3, dt=dt)
        x[:, :64] = 0
        x[:, 0] = x[:, 16] = 4.0
        x[:, 32] = x[:, 48] = level / 4
        conv = torch.ones(1, C)
        want = attn_oracle(x, conv, sh)
        no_sink = want / (1 - 1 / (1 + (torch.arange(1, T + 1)[:, None]) * np.exp(level)))
        if level < 5:
            assert (no_sink - want).abs().max() > 0.05
        y = hops.sink_attention(x.to(dev), conv.to(dev), cos, sin, sh, hops.PromptRows([T], dev), 0)
        close(y, want, dt)


def test_rotation_tables_far_positions():
    """cos / sin of large positions to f32 rounding of the exact angle."""
    cos, sin = hops.pair_rope_tables(100001, 8, 5e4)
    for p in (0, 1, 4097, 100000):
        for i in range(4):
            a = p * 5e4 ** (-2 * i / 8)
            assert abs(float(cos[p, i]) - np.cos(a)) < 1e-6 and abs(float(sin[p, i]) - np.sin(a)) < 1e-6


# ------------------------------------------------------------------ whole models
A, M = orc.attention, orc.mingru
CONFIGS = {
    "mixed": orc.config(48, 301, 3, [M(80, 96), A(4, 2, 16, 16, 4, 24, 1e4, 8, 0.25, 72), A(2, 1, 20, 12, 3, 10, 3e3, 20, 0.3),
                                     M(33)], eps=1e-4),
    "attention_only": orc.config(40, 97, 1, [A(3, 3, 24, 32, 2, 9, 1e5, 4, 0.2, 56), A(6, 2, 8, 8, 1, 300, 1e4, 0, 0.35, 40)]),
    "mingru_only": orc.config(36, 64, 4, [M(20), M(64, 30)]),
    "wide_heads": orc.config(64, 128, 8, [A(2, 1, 144, 80, 4, 33, 2e4, 64, 0.08, 64), M(64, 64)]),
    "long_chunk": orc.config(32, 80, 2, [M(32), A(4, 1, 32, 32, 4, 600, 1e4, 16, 0.2, 64)]),
    # widths the fused decode kernels take (multiples of 512), padded heads, four-channel tails
    "fused": orc.config(512, 128, 4, [M(68, 512), A(4, 2, 36, 20, 3, 21, 1e4, 12, 0.2, 1024), M(512)]),
}


@pytest.fixture(scope="module")
def built(tmp_path_factory):
    cache = {}

    def get(name, dev, dt):
        if name not in cache:
            cfg = CONFIGS[name]
            w = orc.random_weights(cfg, seed=sum(map(ord, name)))
            cache[name] = (cfg, w, orc.save(cfg, w, tmp_path_factory.mktemp(name)))
        cfg, w, path = cache[name]
        return cfg, w, build_model(path, device=dev, dtype=dt)

    return get


def tokens(n, vocab, seed):
    return torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def logits_close(got, want, dt):
    """Mean-free RMS difference of every row against the spread of the logits."""
    d = got.double().cpu() - want.double()
    d = (d - d.mean(-1, keepdim=True)).pow(2).mean(-1).sqrt() / want.double().std(-1).mean()
    assert float(d.max()) < (1e-4 if dt == torch.float32 else 6e-2), float(d.max())


@on_devices
@pytest.mark.parametrize("name", list(CONFIGS))
def test_model_prompts_then_decoding(built, name, dev, dt):
    """Logits of every position: whole prompts of unequal length in one pass, then decoded together past
    several chunk edges, against the oracle and against each request alone."""
    cfg, w, model = built(name, dev, dt)
    V, lens, more = cfg["vocab"], [5, 1, 30, 12], 24
    if name == "long_chunk":
        lens, more = [560, 3, 255, 1], 50
    seqs = [tokens(n + more, V, 50 + i) for i, n in enumerate(lens)]
    want = [orc.forward(cfg, w, s, torch.float32) for s in seqs]
    eng = Engine(model, max_batch=6, max_seq=1024, kv_pool_tokens=6 * 1024)
    slots = [eng.acquire() for _ in lens]
    for s, n in zip(slots, lens):
        eng.extend(s, n + 1)
    got = eng.prefill_batch(slots, [s[:n] for s, n in zip(seqs, lens)], [list(range(n)) for n in lens])
    logits_close(got, torch.cat([x[:n] for x, n in zip(want, lens)]), dt)
    for t in range(more):
        for s, n in zip(slots, lens):
            eng.extend(s, n + t + 1)
        lg = eng.decode(slots, torch.tensor([s[n + t] for s, n in zip(seqs, lens)])).float().clone()
        logits_close(lg, torch.stack([x[n + t] for x, n in zip(want, lens)]), dt)
    for s in slots:
        eng.release(s)
    # each alone in the slots and blocks just given back, shorter, one token at a time from the first
    for s in seqs[:2]:
        slot = eng.acquire()
        eng.extend(slot, 40)
        ref = orc.forward(cfg, w, s[:20], torch.float32)
        out = [eng.prefill_batch([slot], [s[:1]])[0]]
        out += [eng.decode([slot], torch.tensor([t]))[0].float().clone() for t in s[1:20]]
        logits_close(torch.stack(out), ref, dt)
        eng.release(slot)


@on_devices
def test_residual_stream_layer_by_layer(built, dev, dt):
    cfg, w, model = built("mixed", dev, dt)
    ids = tokens(31, cfg["vocab"], 3)
    want, got = [], []
    orc.forward(cfg, w, ids, torch.float64, want)
    model.hidden_states(torch.tensor([ids], device=dev), tap=lambda i, h: got.append(h.clone()))
    assert len(got) == len(want) == len(cfg["layers"])
    for a, b in zip(got, want):
        close(a, b, dt, 2)


@pytest.mark.parametrize("dev", ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)])
@pytest.mark.parametrize("name", ["mixed", "mingru_only", "attention_only"])
def test_greedy_generation_through_the_scheduler(built, name, dev):
    """More requests than slots, unequal prompts and lengths, a pool that makes some wait; f32."""
    cfg, w, model = built(name, dev, torch.float32)
    prompts = [tokens(n, cfg["vocab"], n) for n in (1, 2, 9, 26, 14, 5)]
    want = [orc.greedy(cfg, w, p, 8, torch.float32) for p in prompts]
    for kw in ({}, {"kv_pool_tokens": 512}, {"prefill_tokens": 12}):
        eng = Engine(model, max_batch=3, max_seq=256, eos_ids=(model.cfg.eos_id,), **kw)
        assert eng.generate(prompts, max_new_tokens=8) == want
        assert eng.generate(prompts[::-1], max_new_tokens=8) == want[::-1]


def test_long_decoding_keeps_a_bounded_cache(built):
    """A slot owns the blocks of one chunk however long its sequence grows."""
    cfg, w, model = built("mixed", "cpu", torch.float32)
    eng = Engine(model, max_batch=2, max_seq=100000, kv_pool_tokens=512)
    assert eng.kv.span == 24 and eng.kv.maxb == 1 and eng.kv.blocks_for(90000) == 1
    seq = tokens(300, cfg["vocab"], 8)
    slot = eng.acquire()
    eng.extend(slot, 100000)
    lg = eng.prefill_batch([slot], [seq[:1]])
    for t in seq[1:]:
        lg = eng.decode([slot], torch.tensor([t]))
    logits_close(lg, orc.forward(cfg, w, seq, torch.float32)[-1:], torch.float32)
    assert len(eng.kv.owned[slot]) == 1


def test_engine_embeddings(built):
    cfg, w, model = built("mixed", "cpu", torch.float32)
    eng = Engine(model, max_batch=2, max_seq=64)
    e = eng.embed([tokens(9, cfg["vocab"], 1), tokens(3, cfg["vocab"], 2)])
    assert e.shape == (2, 48) and torch.allclose(e.norm(dim=1), torch.ones(2), atol=1e-5)


def test_engine_rejects_bad_tokens(built):
    _, _, model = built("mixed", "cpu", torch.float32)
    eng = Engine(model, max_batch=2, max_seq=64)
    for bad in ([], [5, 301], [-1]):
        with pytest.raises(ValueError):
            eng.prefill_batch([0], [bad])


def test_tensor_parallel_and_lora_are_refused(built):
    _, _, model = built("mixed", "cpu", torch.float32)
    with pytest.raises(NotImplementedError):
        Revesun(model.cfg, lora_r=4)


# ------------------------------------------------------------------ configuration, weights, command line
def test_config_round_trip_and_errors(tmp_path):
    cfg = CONFIGS["mixed"]
    c = RevesunConfig.from_json(cfg)
    assert c.to_json() == cfg and c.n_layers == 4 and RevesunConfig.from_json(c.to_json()) == c
    assert c.n_params() == sum(int(np.prod(s)) for s in orc.tensor_shapes(cfg).values())
    for change in ({"type": "other"}, {"mlp": {"kind": "sparse", "ff": 8}},
                   {"mixer": dict(cfg["layers"][1]["mixer"], kv_heads=3)},
                   {"mixer": dict(cfg["layers"][1]["mixer"], rot={"base": 1e4, "dims": 7})}):
        bad = json.loads(json.dumps(cfg))
        bad["layers"][1].update(change)
        with pytest.raises(ValueError):
            RevesunConfig.from_json(bad)
    (tmp_path / "config.json").write_text(json.dumps(dict(cfg, architecture="Nothing")))
    with pytest.raises(ValueError):
        model_config(str(tmp_path))


def test_weights_round_trip_and_strictness(tmp_path):
    cfg = CONFIGS["mixed"]
    w = orc.random_weights(cfg, 5)
    m = build_model(orc.save(cfg, w, tmp_path / "a"), dtype=torch.float32)
    assert sum(p.numel() for p in m.parameters()) == m.cfg.n_params()
    save_revesun(m, str(tmp_path / "b"))
    m2 = build_model(str(tmp_path / "b"), dtype=torch.float32)
    for (n, p), (_, q) in zip(m.named_parameters(), m2.named_parameters()):
        assert torch.equal(p, q), n
    for name, change in (("missing", lambda d: d.pop("l1.mix.k.conv")),
                         ("extra", lambda d: d.update({"l9.norm1": torch.ones(3)})),
                         ("shape", lambda d: d.update({"l1.mix.q": torch.zeros(64, 40)}))):
        d = dict(w)
        change(d)
        with pytest.raises((KeyError, ValueError)):
            build_model(orc.save(cfg, d, tmp_path / name))


def test_presets_build_and_serve():
    m = build_model("revesun-tiny", dtype=torch.float32, seed=3)
    assert isinstance(m, Revesun) and m.num_params() == m.cfg.n_params()
    out = Engine(m, max_batch=2, max_seq=128).generate([[1, 2, 3], [9]], max_new_tokens=5)
    assert [len(o) for o in out] == [5, 5]


def test_server_serves_a_model_directory(tmp_path):
    """The HTTP server's engine builder takes a Revesun directory like any other model."""
    from mxllm.serve.server import build_default

    cfg = orc.config(24, 300, 2, [M(16), A(2, 1, 8, 8, 2, 12, 1e4, 4, 0.3, 16)])
    eng, tok = build_default(orc.save(cfg, orc.random_weights(cfg, 1), tmp_path), device="cpu", max_batch=2, max_seq=128)
    ids = tok.encode("hello")
    assert max(ids) < 300 and len(eng.generate([ids], max_new_tokens=4)[0]) == 4


@pytest.mark.parametrize("dev", ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)])
def test_trace_replay(built, dev, tmp_path):
    """JSON steps in, logits files out: batches, finished requests, ids used again, nothing wanted."""
    from mxllm.serve.trace import Replay, replay

    cfg, w, model = built("mixed", dev, torch.float32)
    seqs = {"a": tokens(40, 301, 1), "b": tokens(12, 301, 2)}
    want = {k: orc.forward(cfg, w, s, torch.float32) for k, s in seqs.items()}
    steps, expect = [], []

    def step(entries, end=()):
        n = len(steps)
        steps.append(json.dumps({"step": n, "entries": [{"id": i, "tokens": seqs[i][lo:hi], "want": wt}
                                                        for i, lo, hi, wt in entries], "end": list(end)}))
        expect.append([want[i][lo + k] for i, lo, hi, wt in entries for k in wt])

    for _ in range(2):
        step([("a", 0, 20, [19, 0, 7]), ("b", 0, 9, [])])
        step([("a", 20, 21, []), ("b", 9, 10, [])])
        for p in range(21, 23):
            step([("b", p - 11, p - 10, [0]), ("a", p, p + 1, [0])])
        step([("a", 23, 24, [0])], ["b"])
        for p in range(24, 32):
            step([("a", p, p + 1, [0] if p % 3 else [])])
        step([("a", 32, 33, [0])], ["a"])
    eng = Engine(model, max_batch=3, max_seq=64, kv_pool_tokens=1024)
    said = []
    replay(eng, io.StringIO("\n".join(steps) + "\n"), str(tmp_path), said.append)
    assert said == [f"done {i}" for i in range(len(steps))]
    for i, rows in enumerate(expect):
        f = tmp_path / f"{i}.f32"
        assert f.exists() == bool(rows)
        if rows:
            logits_close(torch.from_numpy(np.fromfile(f, dtype="<f4").reshape(len(rows), 301)), torch.stack(rows),
                         torch.float32)
    assert sorted(eng.free_slots) == [0, 1, 2] and not Replay(eng).slot


def test_trace_refuses_float32_where_kernels_are_bf16(tmp_path, capsys):
    from mxllm.serve import trace

    (tmp_path / "config.json").write_text(json.dumps({
        "model_type": "llama", "vocab_size": 64, "hidden_size": 32, "num_hidden_layers": 1, "num_attention_heads": 2,
        "intermediate_size": 64}))
    assert trace.main(["--model", str(tmp_path), "--dtype", "float32", "--out", str(tmp_path), "--max-tokens", "8"]) == 3


def test_kvcache_span_and_growth():
    kv = KVCache(0, 0, 0, torch.float32, torch.device("cpu"), 3, 4096, pool_tokens=1024, shapes=[(1, 8, 16), (2, 4, 4)],
                 span=600)
    assert [tuple(k.shape[1:]) for k in kv.k] == [(1, 256, 8), (2, 256, 4)] and kv.v[0].shape[3] == 16
    assert kv.maxb == 3 and kv.blocks_for(5000) == 3 and kv.capacity(0) == 0
    kv.grow(0, 10)
    first = kv.owned[0][0]
    kv.k[0][first, 0, 3] = 7
    kv.grow(1, 300)
    kv.grow(0, 257)
    assert kv.owned[0][0] == first and kv.capacity(0) == 512 and len(kv.free) == 0
    kv.grow(0, 500)  # already held
    with pytest.raises(RuntimeError):
        kv.grow(1, 600)
    kv.release(1)
    kv.grow(0, 3000)
    assert kv.capacity(0) == 4096 and kv.bt_host[0].tolist() == kv.owned[0]
    assert float(kv.k[0][first, 0, 3, 0]) == 7


# ------------------------------------------------------------------ GPU only
@pytest.mark.gpu
@pytest.mark.parametrize("batch", [1, 2, 5, 8])
def test_fused_decode_equals_its_parts(built, gpu, batch, monkeypatch):
    """The fused decode kernels against the separate ones on the same steps, and graph replays against
    eager steps, with the same slots and blocks."""
    cfg, w, model = built("fused", gpu, torch.bfloat16)
    prompts = [tokens(3 + 4 * i, 128, i) for i in range(batch)]
    feed = torch.randint(0, 128, (50, batch), generator=torch.Generator().manual_seed(1))
    outs = []
    for fused, graphs in ((True, True), (True, False), (False, False)):
        monkeypatch.setattr(hops, "FUSED", fused)
        eng = Engine(model, max_batch=8, max_seq=256, use_graphs=graphs, kv_pool_tokens=4096)
        slots = [eng.acquire() for _ in prompts]
        for s, p in zip(slots, prompts):
            eng.extend(s, len(p) + 60)
        eng.prefill_batch(slots, prompts)
        outs.append(torch.stack([eng.decode(slots, t).float().clone() for t in feed]))
    # the batch is padded to a graph bucket: same kernels or the next ones, so equal up to rounding
    for o in outs[1:]:
        rel = (outs[0] - o).pow(2).mean().sqrt() / o.pow(2).mean().sqrt()
        assert float(rel) < 1.5e-2, float(rel)
    ref = torch.stack([orc.forward(cfg, w, p + feed[:, i].tolist(), torch.float32)[len(p):]
                       for i, p in enumerate(prompts[:2])], 1)
    logits_close(outs[0][:, :2], ref, torch.bfloat16)


@pytest.mark.gpu
def test_fp8_weights_serve(built, gpu):
    """Quantised projections take the unfused steps; the logits stay near the bf16 model's."""
    from mxllm.serve.quant import quantize_model_fp8_

    _, _, model = built("fused", gpu, torch.bfloat16)
    seq = tokens(40, 128, 4)
    ref = Engine(model, max_batch=2, max_seq=128).prefill_batch([0], [seq], [[39]])
    assert quantize_model_fp8_(model) > 0
    eng = Engine(model, max_batch=2, max_seq=128)
    eng.prefill_batch([0], [seq[:39]])
    got = eng.decode([0], torch.tensor([seq[39]])).float()
    rel = (got - ref).pow(2).mean().sqrt() / ref.pow(2).mean().sqrt()
    assert float(rel) < 0.2, float(rel)


@pytest.mark.gpu
def test_bf16_generation_matches_its_own_prompt_pass(built, gpu):
    """Greedy bf16 generation through the scheduler: every chosen token is the argmax of the prompt pass over
    the same tokens, up to near-ties."""
    cfg, _, model = built("mixed", gpu, torch.bfloat16)
    prompts = [tokens(n, 301, n) for n in (3, 40, 11, 1, 25)]
    outs = Engine(model, max_batch=4, max_seq=256).generate(prompts, max_new_tokens=40)
    for p, o in zip(prompts, outs):
        lg = model(torch.tensor([p + o[:-1]], device=gpu))[0, len(p) - 1:].float()
        top = lg.max(-1).values
        got = lg.gather(1, torch.tensor(o, device=gpu)[:, None])[:, 0]
        assert float((top - got).max()) < 0.05 * float(lg.std())
