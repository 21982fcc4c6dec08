"""Helpers of the whole-model tests of model-folder designs."""
import numpy as np

import mixed_model as mm

# differences of logits: root mean square over root mean square
LIMIT = {"fp32": 2e-5, "bf16": 2.5e-2}


class Case:
    """A configuration, its weights in a folder, and what a plain statement
    (`forward`) says about some tokens."""

    def __init__(self, config, weights, forward, folder, tokens=210):
        self.config, self.weights, self.forward = config, weights, forward
        self.path = mm.write_folder(folder, config, weights)
        self.tokens = np.random.default_rng(4).integers(0, config["vocab"], tokens)
        self.logits, self.streams = self.expect(self.tokens)

    def expect(self, tokens):
        return self.forward(self.config, mm.float64(self.weights), tokens)


def distance(got, want):
    got, want = np.asarray(got, np.float64), np.asarray(want, np.float64)
    return np.sqrt(np.mean((got - want) ** 2, axis=-1) / np.mean(want ** 2))


def feed(model, request, tokens, counts):
    """Logits of every position, the tokens cut into portions of these sizes
    (the last one repeated)."""
    out, at = [], 0
    for index in range(len(tokens)):
        count = min(counts[min(index, len(counts) - 1)], len(tokens) - at)
        logits, _ = model.step(request, tokens[at:at + count], range(count))
        out.append(logits)
        at += count
        if at == len(tokens):
            break
    return np.concatenate(out)


def continuation(case, prompt, count):
    """Greedy tokens of the plain statement, and how close its choices were."""
    tokens, margins = list(prompt), []
    for _ in range(count):
        row = case.expect(tokens)[0][-1]
        top = np.sort(row)[-2:]
        margins.append(top[1] - top[0])
        tokens.append(int(row.argmax()))
    return tokens[len(prompt):], min(margins)
