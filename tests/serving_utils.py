"""Helpers of the serving tests: where they run, ragged batches for single ops, portions of sequences, comparisons."""
import types

import pytest
import torch

GPU = pytest.mark.gpu
RUNS = [pytest.param(("cpu", torch.float32), id="cpu"),
        pytest.param(("cuda", torch.float32), id="gpu-f32", marks=GPU),
        pytest.param(("cuda", torch.bfloat16), id="gpu-bf16", marks=GPU)]


@pytest.fixture(params=RUNS)
def run(request):
    dev, dtype = request.param
    if dev == "cuda" and not torch.cuda.is_available():
        pytest.skip("no GPU")
    print(f"[{request.node.name}]", flush=True)
    return torch.device(dev), dtype


def tol(dtype, f32=2e-5, bf16=2e-2):
    return f32 if dtype == torch.float32 else bf16


def close(got, want, dtype, f32=2e-5, bf16=2e-2):
    """Root mean square error relative to the wanted values' root mean square, worst row."""
    got, want = got.double().cpu(), want.double().cpu()
    assert got.shape == want.shape
    assert torch.isfinite(got).all()
    if got.numel() == 0:
        return
    err = (got - want).reshape(got.shape[0], -1).pow(2).mean(-1).sqrt().max()
    ref = want.pow(2).mean().sqrt()
    assert err <= tol(dtype, f32, bf16) * ref, (float(err / ref), got.shape)


# -----------------------------------------------------------------------------------------------
# batches for the ops: sequences with (new tokens, tokens seen), pages handed out in a scrambled order
# -----------------------------------------------------------------------------------------------
class Pages:
    def __init__(self, n_slots, n_blocks, block_size, width, slots, device, dtype):
        g = torch.Generator().manual_seed(5)
        self.bs, self.device, self.slots = block_size, device, slots
        per = n_blocks // n_slots
        perm = torch.randperm(per * n_slots, generator=g).view(n_slots, per)
        self.tables = perm.to(torch.int32)
        self.cache = torch.full((per * n_slots, block_size, width), 3.0, dtype=dtype, device=device)

    def batch(self, seqs):
        """seqs: (sequence number, new tokens, seen)."""
        b = types.SimpleNamespace()
        meta, ts, tp, q0 = [], [], [], 0
        for i, (s, n, seen) in enumerate(seqs):
            meta.append((q0, n, seen))
            ts += [i] * n
            tp += range(seen, seen + n)
            q0 += n
        i32 = lambda v: torch.tensor(v, dtype=torch.int32, device=self.device)  # noqa: E731
        b.seq_meta_host, b.current_tokens, b.current_sequences = meta, q0, len(seqs)
        b.seq_meta, b.tok_seq, b.tok_pos = i32(meta).view(-1, 3), i32(ts), i32(tp)
        b.block_tables = torch.stack([self.tables[s] for s, _, _ in seqs]).to(self.device).contiguous()
        b.slots_host = [self.slots[s] for s, _, _ in seqs]
        b.slots, b.max_new, b.plans = i32(b.slots_host), max(n for _, n, _ in seqs), {}
        b.carry = {}
        return b


def portions(lengths, sizes, seed=0):
    """Steps that feed sequences of these lengths in portions of ``sizes`` (cycled), several sequences a step."""
    g = torch.Generator().manual_seed(seed)
    pos, k, steps = [0] * len(lengths), 0, []
    while any(p < n for p, n in zip(pos, lengths)):
        step = []
        for s, n in enumerate(lengths):
            if pos[s] >= n or (len(step) and torch.rand(1, generator=g) < 0.3):
                continue
            c = min(sizes[k % len(sizes)], n - pos[s])
            k += 1
            step.append((s, c, pos[s]))
            pos[s] += c
        steps.append(step)
    return steps


def rnd(*shape, seed, scale=1.0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed), dtype=torch.float64) * scale


def tokens(vocab, n, seed):
    return torch.randint(0, vocab, (n, ), generator=torch.Generator().manual_seed(seed)).tolist()


def feed(eng, seqs, steps):
    """seqs: token lists; steps: [(sequence, new tokens, position)]. Returns every sequence's logits at all places."""
    outs = [[] for _ in seqs]
    for step in steps:
        lg, _ = eng.put([s for s, _, _ in step], [torch.tensor(seqs[s][p:p + n]) for s, n, p in step],
                        capture_latents=False, logits_at=[range(n) for _, n, _ in step])
        o = 0
        for s, n, _ in step:
            outs[s].append(lg[o:o + n].double().cpu())
            o += n
    return [torch.cat(o) for o in outs]
