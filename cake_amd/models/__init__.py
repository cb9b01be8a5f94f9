"""Model families: Llama-3 and hybrid-design text generation, Stable Diffusion images."""
