"""Model families on the hot path: llama (incl. mistral), qwen3, runevik and dolurax (``utils._get_classes``)."""
