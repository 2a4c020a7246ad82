"""Model families on the hot path: llama (incl. mistral), qwen3, runevik, dolurax, temetar and beronex (``utils._get_classes``)."""
