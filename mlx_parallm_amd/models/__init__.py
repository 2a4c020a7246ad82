"""Model families on the hot path: llama (incl. mistral), qwen3, runevik, dolurax and temetar (``utils._get_classes``)."""
