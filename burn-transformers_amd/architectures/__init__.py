"""Importing this package registers the architectures the library ships (GPT-2, Salopel, Kodatar, Rotutar, Gavasun,
Loselix, Rirovik)."""

from . import gavasun, gpt2, kodatar, loselix, rirovik, rotutar, salopel  # noqa: F401
