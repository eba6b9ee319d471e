"""Token choice from a batch of logits, shared by the inference engines."""
import torch


def sample_tokens(logits, do_sample=False, temperature=1.0, top_k=0, top_p=1.0, generator=None):
    """logits [B, V] -> token ids [B]: greedy, or temperature / top-k / nucleus sampling."""
    if not do_sample:
        return logits.argmax(-1)
    logits = logits.float() / max(temperature, 1e-5)
    if top_k and top_k > 0:
        kth = torch.topk(logits, min(top_k, logits.shape[-1]), dim=-1).values[..., -1:]
        logits = logits.masked_fill(logits < kth, float("-inf"))
    if top_p is not None and top_p < 1.0:
        srt, idx = torch.sort(logits, descending=True, dim=-1)
        cum = srt.softmax(-1).cumsum(-1)
        drop = cum - srt.softmax(-1) > top_p
        srt = srt.masked_fill(drop, float("-inf"))
        logits = torch.full_like(logits, float("-inf")).scatter(-1, idx, srt)
    probs = logits.softmax(-1)
    return torch.multinomial(probs, 1, generator=generator).squeeze(-1)
