"""What the tests of models in folder form share."""
import numpy as np


def errors(got, want):
    """rms error of each position's logits over the deviation of all of them"""
    return np.sqrt(((got - want) ** 2).mean(axis=-1)) / want.std()


def portions(m, tokens, sizes):
    """Logits at every place, fed in portions of the given sizes (the last one repeats); one token is a decode step."""
    m.set_past_len(0)
    out, at, k = [], 0, 0
    while at < len(tokens):
        n = min(sizes[min(k, len(sizes) - 1)], len(tokens) - at)
        if n == 1:
            m.step(tokens[at])
            out.append(m.logits()[None])
        else:
            out.append(m.prefill_logits(tokens[at:at + n], range(n)))
        at, k = at + n, k + 1
    return np.concatenate(out)
