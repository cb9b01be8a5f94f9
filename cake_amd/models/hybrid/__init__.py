"""Hybrid decoder designs: attention and gated-delta layers, optionally looped."""
