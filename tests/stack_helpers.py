"""What the GPU tests of the config-driven stacks share."""
import torch

DT = {"f32": torch.float32, "bf16": torch.bfloat16}


def rnd(*shape, seed=0, scale=1.0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed), dtype=torch.float64) * scale


def relerr(got, want):
    return float((got.double().cpu() - want).abs().max() / (want.abs().max() + 1e-30))


def act(t, ld, dt, rows=None):
    """t [n, k] as an activation buffer of `ld` columns, padding zero."""
    b = torch.zeros(rows or t.shape[0], ld, dtype=dt, device="cuda")
    b[:t.shape[0], :t.shape[1]] = t.to(dt)
    return b


def st():
    return torch.cuda.current_stream().cuda_stream


def run_rows(m, b, kc, state, parts, bs=16):
    """One forward of [(state slot, blocks, first position, tokens)] with every row's logits; CPU logits per part."""
    T = 0
    b.slot.fill_(-1)
    dev = b.ids.device
    for r, (slot, blocks, p0, toks) in enumerate(parts):
        n = len(toks)
        pos = torch.arange(p0, p0 + n)
        blk = torch.tensor(blocks)
        b.ids[T:T + n] = torch.tensor(toks, dtype=torch.int32)
        b.pos[T:T + n] = pos.int()
        b.slot[T:T + n] = (blk[pos // bs] * bs + pos % bs).int()
        b.tok_seq[T:T + n] = r
        b.ctx_len[T:T + n] = (pos + 1).int()
        b.block_tables[r, :len(blocks)] = blk.int()
        b.runs[r] = torch.tensor([T, n, slot, p0])
        T += n
    qb = m.attention_blocks(b, T)
    rows = torch.arange(T, dtype=torch.int32, device=dev)
    m.forward(b, kc, None, T, bs, logit_rows=rows, n_logits=T, state=state, nruns=len(parts), **qb)
    lg = b.logits[:T].cpu()
    out, o = [], 0
    for _, _, _, toks in parts:
        out.append(lg[o:o + len(toks)])
        o += len(toks)
    return out


def engine(m, **kw):
    from nats_llm_studio_amd.engine.engine import Engine
    kw = dict(dict(max_batch=4, num_blocks=64, max_prefill_tokens=512, max_logit_rows=512, ctx=512), **kw)
    return Engine(m, None, **kw)
