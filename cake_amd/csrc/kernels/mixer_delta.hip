// Gated delta rule of the hybrid designs: a short causal convolution + SiLU on q, k and v,
// unit-norm queries and keys, and per head the recurrence
//     S <- decay S;   u = beta (v - S^T k);   S <- S + k u^T;   o = S^T q
// over a [dim x vdim] state in 32-bit floats, then a gated RMS norm of o.
//
// State of one layer run: S [slot][H][dim][EP] f32 (EP = vdim padded to 4) and a ring of the
// last `taps` raw projections per channel, [slot][taps][C] f32 (C = 2 G dim + H vdim; the
// entry of position p is p % taps, so a token's own entry is never one another workgroup of
// the same step still reads).  A sequence at position 0 starts from zeros whatever its slot
// held before.
//
// Prompt rows run in chunks of 16 tokens.  Inside a chunk (decay products G_ij over tokens
// j+1..i, g_i from the chunk's start), with the chunk's entry state S0:
//     (I + A) U = R,  A_ij = beta_i G_ij (k_i.k_j) for j < i,  R_i = beta_i (v_i - g_i S0^T k_i)
//     o_i = g_i S0^T q_i + sum_{j <= i} G_ij (q_i.k_j) u_j
//     S   = g_15 S0 + sum_j G_15,j k_j u_j^T
// so everything is 16-row f32 matrix products (v_mfma_f32_16x16x4_f32) except the small
// triangular inverse, which does not depend on the state.
//
//   * mixer_delta_prep: convolution, SiLU and unit norms of a chunk's rows.
//   * mixer_delta_chunk: per chunk and head T = (I + A)^-1, P_ij = G_ij (q_i.k_j), g, beta.
//   * mixer_delta_scan: walks the chunks of one sequence.  A workgroup takes 16 columns of one
//     head's S; its four waves hold a quarter of the rows each, as accumulators that are the
//     next chunk's B operands; the partial S0^T k, S0^T q meet in LDS once per chunk.
//   * mixer_delta_out: gated norm of the read-outs.
//   * mixer_delta_decode: all of it for one token per sequence in one launch.
#include "mixer_common.h"

namespace cake {

struct DeltaArgs {
  const void* proj;       // [N][ldp] q | k | v | gate columns (storage type; decode: f32)
  long long ldp;
  const float* ab;        // [N][ldab]: a (H) then b (H)
  long long ldab;
  int N, H, G, dim, vdim, EP, taps;
  float eps;              // read-out norm
  const float* conv;      // [taps][C] f32
  const float* a_log;     // [H] f32
  const float* dt_bias;   // [H] f32
  const float* norm_w;    // [vdim] f32
  int DR;                 // dim padded to 64
  float* qn;              // [N + 15][G][DR], zeros past dim
  float* kn;              // [N + 15][G][DR]
  float* vv;              // [N + 15][H][vdim]
  float* tp;              // [NC][H][2][16][16]: T, P
  float* gm;              // [NC][H][4][16]: g_i, beta_i, G_15,i, g_15
  float* o;               // [N][H][vdim]
  float* state;
  float* ring;
  long long s_slot, r_slot;
  const int* row_pos;     // [N]
  const int* row_slot;    // [N]
  const int* row_seq0;    // [N] packed row of the sequence's first token in this step
  const SeqRow* seq;      // [B]
  const int2* chunk;      // [NC]: packed row of the first token, tokens
  const int* chunk0;      // [B]: first chunk of the sequence
  int NC;
  void* out;              // [N][ldo]
  long long ldo;
};

__device__ __forceinline__ int delta_channels(const DeltaArgs& a) {
  return 2 * a.G * a.dim + a.H * a.vdim;
}

// the raw projection of channel c, `back` tokens before packed row n at position pos
template <int DT>
__device__ __forceinline__ float conv_tap(const DeltaArgs& a, int n, int pos, int first, int back,
                                          int c, const float* ring, int C) {
  if (pos < back) return 0.f;
  if (n - back >= first)
    return St<DT>::ld(reinterpret_cast<const typename St<DT>::E*>(a.proj)[(long long)(n - back) *
                                                                             a.ldp + c]);
  return ring[(long long)((pos - back) % a.taps) * C + c];
}

constexpr int kChunk = 16;

// A wave per (chunk, unit): units [0, 2G) the q and k heads, [2G, 2G + H) the value heads;
// CPL consecutive channels per lane, the last kWin inputs of each in registers (longer
// convolutions read the older ones from memory).
template <int DT, int CPL, int kWin>
__global__ __launch_bounds__(256) void mixer_delta_prep_kernel(DeltaArgs a, int vec) {
  using E = typename St<DT>::E;
  const int lane = threadIdx.x & 63;
  const int units = 2 * a.G + a.H;
  const long long item = (long long)blockIdx.x * 4 + (threadIdx.x >> 6);
  if (item >= (long long)a.NC * units) return;
  const int ch = (int)(item / units), u = (int)(item - (long long)ch * units);
  const int C = delta_channels(a);
  const int n0 = a.chunk[ch].x, cnt = a.chunk[ch].y;
  const int pos0 = a.row_pos[n0], first = a.row_seq0[n0];
  const float* ring = a.ring + a.row_slot[n0] * a.r_slot;
  const bool isv = u >= 2 * a.G;
  const int size = isv ? a.vdim : a.dim;
  const int cb = isv ? 2 * a.G * a.dim + (u - 2 * a.G) * a.vdim : u * a.dim;
  const int c0 = CPL * lane;
  float* out = isv ? a.vv + (u - 2 * a.G) * a.vdim
                   : (u < a.G ? a.qn + u * a.DR : a.kn + (u - a.G) * a.DR);
  const long long ostride = isv ? (long long)a.H * a.vdim : (long long)a.G * a.DR;
  const int osize = isv ? a.vdim : a.DR;
  const float qs = u < a.G ? 1.f / sqrtf((float)a.dim) : 1.f;

  float w[kWin][CPL], win[kWin][CPL];
#pragma unroll
  for (int j = 0; j < kWin; ++j)
#pragma unroll
    for (int e = 0; e < CPL; ++e) {
      const bool ok = j < a.taps && c0 + e < size;
      w[j][e] = ok ? a.conv[(long long)(a.taps - 1 - j) * C + cb + c0 + e] : 0.f;
      // input j tokens before row 0 lives at index (0 - j) & 7
      win[(kWin - j) & (kWin - 1)][e] =
          ok && j > 0 ? conv_tap<DT>(a, n0, pos0, first, j, cb + c0 + e, ring, C) : 0.f;
    }
  const E* src = reinterpret_cast<const E*>(a.proj) + (long long)n0 * a.ldp + cb + c0;
#pragma unroll
  for (int t = 0; t < kChunk; ++t) {
    if (t < cnt) {  // wave-uniform
      float x[CPL];
      if constexpr (CPL == 2 && DT != kF32) {
        if (vec && c0 + 1 < size) {
          const uint32_t p = *reinterpret_cast<const uint32_t*>(src + (long long)t * a.ldp);
          x[0] = St<DT>::ld((uint16_t)(p & 0xffffu));
          x[1] = St<DT>::ld((uint16_t)(p >> 16));
        } else {
#pragma unroll
          for (int e = 0; e < CPL; ++e)
            x[e] = c0 + e < size ? St<DT>::ld(src[(long long)t * a.ldp + e]) : 0.f;
        }
      } else {
#pragma unroll
        for (int e = 0; e < CPL; ++e)
          x[e] = c0 + e < size ? St<DT>::ld(src[(long long)t * a.ldp + e]) : 0.f;
      }
      float y[CPL], ss = 0.f;
#pragma unroll
      for (int e = 0; e < CPL; ++e) {
        win[t & (kWin - 1)][e] = x[e];
        y[e] = 0.f;
#pragma unroll
        for (int j = 0; j < kWin; ++j) y[e] = fmaf(w[j][e], win[(t - j) & (kWin - 1)][e], y[e]);
        if (a.taps > kWin)  // longer convolutions: the older inputs from memory
          for (int j = kWin; j < a.taps; ++j)
            if (c0 + e < size)
              y[e] = fmaf(a.conv[(long long)(a.taps - 1 - j) * C + cb + c0 + e],
                          conv_tap<DT>(a, n0 + t, pos0 + t, first, j, cb + c0 + e, ring, C), y[e]);
        y[e] = silu32(y[e]);
        ss += y[e] * y[e];
      }
      const float r = isv ? 1.f : qs / sqrtf(wave_sum(ss) + 1e-6f);
      float* o = out + (long long)(n0 + t) * ostride + c0;
      if constexpr (CPL == 2) {
        if (c0 + 1 < osize && (osize & 1) == 0) {
          *reinterpret_cast<float2*>(o) = make_float2(y[0] * r, y[1] * r);
          continue;
        }
      }
#pragma unroll
      for (int e = 0; e < CPL; ++e)
        if (c0 + e < osize) o[e] = y[e] * r;
    } else if (n0 + cnt == a.N) {  // the scan reads whole chunks: zeros past the last row
      for (int e = 0; e < CPL; ++e)
        if (c0 + e < osize) out[(long long)(n0 + t) * ostride + c0 + e] = 0.f;
    }
  }
}

// A wave per (chunk, kv head): the state-independent matrices of every head of the group
__global__ __launch_bounds__(256) void mixer_delta_chunk_kernel(DeltaArgs a) {
  __shared__ float kks[4][16][17], qks[4][16][17], ams[4][4][16][17];
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, l15 = lane & 15, g = lane >> 4;
  const long long item = (long long)blockIdx.x * 4 + wave;
  if (item >= (long long)a.NC * a.G) return;  // waves share nothing
  const int ch = (int)(item / a.G), gh = (int)(item - (long long)ch * a.G);
  const int n0 = a.chunk[ch].x, cnt = a.chunk[ch].y;
  float(&kk)[16][17] = kks[wave];
  float(&qk)[16][17] = qks[wave];
  float(&am)[4][16][17] = ams[wave];
  {  // k.k and q.k: rows past the chunk's end repeat the last, masked below
    const int row = n0 + min(l15, cnt - 1);
    const float* kp = a.kn + ((long long)row * a.G + gh) * a.DR + 4 * g;
    const float* qp = a.qn + ((long long)row * a.G + gh) * a.DR + 4 * g;
    cf32x4 ka{0.f, 0.f, 0.f, 0.f}, qa{0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
    for (int d = 0; d < a.DR; d += 16) {  // DR % 64 == 0: four pieces of each in flight
      const uint4 kv = *reinterpret_cast<const uint4*>(kp + d);
      ka = mm_piece<kF32>(kv, kv, ka);
      qa = mm_piece<kF32>(*reinterpret_cast<const uint4*>(qp + d), kv, qa);
    }
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      kk[4 * g + e][l15] = ka[e];
      qk[4 * g + e][l15] = qa[e];
    }
  }
  __builtin_amdgcn_wave_barrier();  // a wave's LDS accesses complete in order
  const int R = a.H / a.G;
  for (int h0 = 0; h0 < R; h0 += 4) {
    // sixteen lanes per head, lane c = column c (and token c)
    const int hs = g, hl = h0 + hs, h = gh * R + min(hl, R - 1), c = l15;
    const bool ok = c < cnt;
    const float* ab = a.ab + (long long)(n0 + min(c, cnt - 1)) * a.ldab;
    const float ld = ok ? fmaxf(-expf(a.a_log[h]) * softplus32(ab[h] + a.dt_bias[h]), -1e30f) : 0.f;
    const float beta = ok ? sigmoid32(ab[a.H + h]) : 0.f;
    float t[16], p[16];
    float s = 0.f, pre = 0.f, suf = 0.f, all = 0.f;
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      const float li = __shfl(ld, 16 * g + i, 64), bi = __shfl(beta, 16 * g + i, 64);
      all += li;
      if (i <= c) pre += li;
      if (i > c) { s += li; suf += li; }
      const float gi = expf(s);  // decay over tokens c + 1 .. i (1 at i = c)
      am[hs][i][c] = i > c ? bi * gi * kk[i][c] : 0.f;
      p[i] = i >= c ? gi * qk[i][c] : 0.f;
    }
    __builtin_amdgcn_wave_barrier();
    // column c of (I + A)^-1 by forward substitution
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      float v = i == c ? 1.f : 0.f;
#pragma unroll
      for (int j = 0; j < i; ++j) v = fmaf(-am[hs][i][j], t[j], v);
      t[i] = v;
    }
    if (hl < R) {
      float* tp = a.tp + ((long long)ch * a.H + h) * 512 + c;
#pragma unroll
      for (int i = 0; i < 16; ++i) { tp[16 * i] = t[i]; tp[256 + 16 * i] = p[i]; }
      float* gp = a.gm + ((long long)ch * a.H + h) * 64 + c;
      gp[0] = expf(pre); gp[16] = beta; gp[32] = expf(suf); gp[48] = expf(all);
    }
    __builtin_amdgcn_wave_barrier();
  }
}

// One chunk's operands of a scan lane.
template <int NI> struct ScanSet {
  u32x4 kp[NI], qp[NI], t, p;
  float kt[NI][4], v[4], g15;
  cf32x4 gi, beta, ge;  // tokens 4 g .. 4 g + 3
};

// grid (H, ceil(vdim / 16), B) — the column blocks of a head land on one XCD and share its
// rows in that L2 — 256 threads; wave w: rows [16 NI w, 16 NI (w + 1)), DR = 64 NI
template <int DT, int NI>
__global__ __launch_bounds__(256) void mixer_delta_scan_kernel(DeltaArgs a) {
  using E = typename St<DT>::E;
  constexpr int DR = 64 * NI;
  __shared__ __attribute__((aligned(16))) float ex[2][4][2][64][4];
  const SeqRow sq = a.seq[blockIdx.z];
  const int h = blockIdx.x, R = a.H / a.G, gh = h / R, c0 = blockIdx.y * 16;
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, l15 = lane & 15, g = lane >> 4;
  const int col = c0 + l15;
  const bool cok = col < a.vdim;
  const int r0 = 16 * NI * wave;
  float* st = a.state + sq.slot * a.s_slot + (long long)h * a.dim * a.EP;
  cf32x4 S[NI];
#pragma unroll
  for (int i = 0; i < NI; ++i)
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int r = r0 + 16 * i + 4 * g + e;
      S[i][e] = sq.pos0 > 0 && cok && r < a.dim ? st[(long long)r * a.EP + col] : 0.f;
    }
  const int nc = (sq.len + kChunk - 1) / kChunk, ch0 = a.chunk0[blockIdx.z];
  // A chunk's operands: a uniform base that moves with the chunk plus a lane offset that does
  // not.  Rows past a sequence's end are another sequence's or zeros (prep) and count nothing:
  // their beta is zero.
  const unsigned krow = (unsigned)a.G * DR, vrow = (unsigned)a.H * a.vdim;
  const unsigned koff = l15 * krow + r0 + 4 * g, toff = 16 * l15 + 4 * g;
  unsigned ktoff[4], voff[4];
#pragma unroll
  for (int e = 0; e < 4; ++e) {
    ktoff[e] = (4 * g + e) * krow + r0 + l15;
    voff[e] = (4 * g + e) * vrow + (cok ? col : 0);
  }
  const float* kbase = a.kn + ((long long)sq.row0 * a.G + gh) * DR;
  const float* qbase = a.qn + ((long long)sq.row0 * a.G + gh) * DR;
  const float* vbase = a.vv + (long long)sq.row0 * vrow + (long long)h * a.vdim;
  const float* tbase = a.tp + ((long long)ch0 * a.H + h) * 512;
  const float* gbase = a.gm + ((long long)ch0 * a.H + h) * 64;
  auto load = [&](ScanSet<NI>& s, int c) __attribute__((always_inline)) {
    const float* kb = kbase + (long long)c * kChunk * krow;
    const float* qb = qbase + (long long)c * kChunk * krow;
    const float* vb = vbase + (long long)c * kChunk * vrow;
    const float* tb = tbase + (long long)c * a.H * 512;
    const float* gb = gbase + (long long)c * a.H * 64;
#pragma unroll
    for (int i = 0; i < NI; ++i) {
      s.kp[i] = *reinterpret_cast<const u32x4*>(kb + koff + 16 * i);
      s.qp[i] = *reinterpret_cast<const u32x4*>(qb + koff + 16 * i);
    }
#pragma unroll
    for (int e = 0; e < 4; ++e) s.v[e] = vb[voff[e]];
    s.gi = *reinterpret_cast<const cf32x4*>(gb + 4 * g);
    s.beta = *reinterpret_cast<const cf32x4*>(gb + 16 + 4 * g);
    s.t = *reinterpret_cast<const u32x4*>(tb + toff);
    s.ge = *reinterpret_cast<const cf32x4*>(gb + 32 + 4 * g);
    s.g15 = gb[48];
#pragma unroll
    for (int i = 0; i < NI; ++i)
#pragma unroll
      for (int e = 0; e < 4; ++e) s.kt[i][e] = kb[ktoff[e] + 16 * i];
    s.p = *reinterpret_cast<const u32x4*>(tb + 256 + toff);
  };
  auto chunk = [&](const ScanSet<NI>& s, int c) __attribute__((always_inline)) {
    const int buf = c & 1;
    cf32x4 ks{0.f, 0.f, 0.f, 0.f}, qs{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int i = 0; i < NI; ++i) {
      const uint4 sb = __builtin_bit_cast(uint4, S[i]);
      ks = mm_piece<kF32>(__builtin_bit_cast(uint4, s.kp[i]), sb, ks);
      qs = mm_piece<kF32>(__builtin_bit_cast(uint4, s.qp[i]), sb, qs);
    }
    *reinterpret_cast<cf32x4*>(ex[buf][wave][0][lane]) = ks;
    *reinterpret_cast<cf32x4*>(ex[buf][wave][1][lane]) = qs;
    // the other waves' halves only need the LDS writes: a full barrier would also drain the
    // operand loads in flight
    asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory");
    ks = *reinterpret_cast<const cf32x4*>(ex[buf][0][0][lane]);
#pragma unroll
    for (int w = 1; w < 4; ++w) ks += *reinterpret_cast<const cf32x4*>(ex[buf][w][0][lane]);
    cf32x4 rhs;
#pragma unroll
    for (int e = 0; e < 4; ++e) rhs[e] = s.beta[e] * (s.v[e] - s.gi[e] * ks[e]);
    const cf32x4 u = mm_piece<kF32>(__builtin_bit_cast(uint4, s.t), __builtin_bit_cast(uint4, rhs),
                                    cf32x4{0.f, 0.f, 0.f, 0.f});
    cf32x4 ud;
#pragma unroll
    for (int e = 0; e < 4; ++e) ud[e] = s.ge[e] * u[e];
    const uint4 ub = __builtin_bit_cast(uint4, ud);
#pragma unroll
    for (int i = 0; i < NI; ++i) {
      const cf32x4 ka = {s.kt[i][0], s.kt[i][1], s.kt[i][2], s.kt[i][3]};
      S[i] = mm_piece<kF32>(__builtin_bit_cast(uint4, ka), ub, S[i] * s.g15);
    }
    if (wave == (c & 3)) {  // the read-outs of a chunk: the waves take turns
      qs = *reinterpret_cast<const cf32x4*>(ex[buf][0][1][lane]);
#pragma unroll
      for (int w = 1; w < 4; ++w) qs += *reinterpret_cast<const cf32x4*>(ex[buf][w][1][lane]);
#pragma unroll
      for (int e = 0; e < 4; ++e) qs[e] *= s.gi[e];
      const cf32x4 o = mm_piece<kF32>(__builtin_bit_cast(uint4, s.p), __builtin_bit_cast(uint4, u), qs);
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int t = kChunk * c + 4 * g + e;
        if (cok && t < sq.len) a.o[((long long)(sq.row0 + t) * a.H + h) * a.vdim + col] = o[e];
      }
    }
  };
  // operands two chunks ahead (chunks past the end re-read the last one)
  ScanSet<NI> s0, s1;
  load(s0, 0);
  load(s1, min(1, nc - 1));
  // once: with loads pending on the way in, the compiler waits for the newest loads in every
  // round (its counts cover both ways into the loop)
  __builtin_amdgcn_s_waitcnt(vm_wait(0));
  for (int c = 0; c < nc; c += 2) {
    chunk(s0, c);
    if (c + 1 >= nc) break;
    load(s0, min(c + 2, nc - 1));
    chunk(s1, c + 1);
    load(s1, min(c + 3, nc - 1));
  }
  if (cok)
#pragma unroll
    for (int i = 0; i < NI; ++i)
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int r = r0 + 16 * i + 4 * g + e;
        if (r < a.dim) st[(long long)r * a.EP + col] = S[i][e];
      }
  // the ring entries of the last taps - 1 tokens (every prompt row has been convolved by now)
  if (blockIdx.y != 0) return;
  const int C = delta_channels(a);
  float* ring = a.ring + sq.slot * a.r_slot;
  const int keep = min(a.taps - 1, sq.len);
  const int nq = h % R == 0 ? 2 * a.dim : 0;  // q and k channels: the group's first head
  for (int i = tid; i < keep * (nq + a.vdim); i += 256) {
    const int j = i / (nq + a.vdim), x = i - j * (nq + a.vdim);
    const int cc = x < nq ? (x < a.dim ? gh * a.dim + x : (a.G + gh) * a.dim + x - a.dim)
                          : 2 * a.G * a.dim + h * a.vdim + x - nq;
    const int row = sq.len - 1 - j;
    ring[(long long)((sq.pos0 + row) % a.taps) * C + cc] =
        St<DT>::ld(reinterpret_cast<const E*>(a.proj)[(long long)(sq.row0 + row) * a.ldp + cc]);
  }
}

// a wave per (row, head): o / rms(o) * norm_w * silu(gate)
template <int DT>
__global__ __launch_bounds__(256) void mixer_delta_out_kernel(DeltaArgs a) {
  using E = typename St<DT>::E;
  const int lane = threadIdx.x & 63;
  const long long item = (long long)blockIdx.x * 4 + (threadIdx.x >> 6);
  if (item >= (long long)a.N * a.H) return;
  const long long n = item / a.H;
  const int h = (int)(item - n * a.H);
  const float* o = a.o + item * a.vdim;
  E* out = reinterpret_cast<E*>(a.out) + n * a.ldo + h * a.vdim;
  const E* gp = reinterpret_cast<const E*>(a.proj) + n * a.ldp + delta_channels(a) + h * a.vdim;
  if constexpr (DT != kF32) {
    // two consecutive channels per lane and access where rows allow it
    if (a.vdim % 2 == 0 && a.ldp % 2 == 0 && a.ldo % 2 == 0 && delta_channels(a) % 2 == 0) {
      float2 x[2];
      float ss = 0.f;
#pragma unroll
      for (int i = 0; i < 2; ++i) {
        const int d = 2 * lane + 128 * i;
        x[i] = d < a.vdim ? *reinterpret_cast<const float2*>(o + d) : make_float2(0.f, 0.f);
        ss += x[i].x * x[i].x + x[i].y * x[i].y;
      }
      const float r = 1.f / sqrtf(wave_sum(ss) / (float)a.vdim + a.eps);
#pragma unroll
      for (int i = 0; i < 2; ++i) {
        const int d = 2 * lane + 128 * i;
        if (d >= a.vdim) continue;
        const uint32_t z = *reinterpret_cast<const uint32_t*>(gp + d);
        const float2 w = *reinterpret_cast<const float2*>(a.norm_w + d);
        const float y0 = x[i].x * r * w.x * silu32(St<DT>::ld((uint16_t)(z & 0xffffu)));
        const float y1 = x[i].y * r * w.y * silu32(St<DT>::ld((uint16_t)(z >> 16)));
        *reinterpret_cast<uint32_t*>(out + d) =
            (uint32_t)St<DT>::st(y0) | ((uint32_t)St<DT>::st(y1) << 16);
      }
      return;
    }
  }
  float x[4], ss = 0.f;
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int d = lane + 64 * i;
    x[i] = d < a.vdim ? o[d] : 0.f;
    ss += x[i] * x[i];
  }
  const float r = 1.f / sqrtf(wave_sum(ss) / (float)a.vdim + a.eps);
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int d = lane + 64 * i;
    if (d < a.vdim) out[d] = St<DT>::st(x[i] * r * a.norm_w[d] * silu32(St<DT>::ld(gp[d])));
  }
}

// One token per sequence, grid (H, B), 512 threads: thread = 4 columns of a few rows of S.
// proj is f32 here.  RPT rows per thread.
constexpr int kDdThreads = 512;
template <int DT, int RPT>
__global__ __launch_bounds__(kDdThreads) void mixer_delta_decode_kernel(DeltaArgs a) {
  using E = typename St<DT>::E;
  __shared__ float q[256], k[256], v[256], u[256];
  __shared__ float red[16], sn[2];
  __shared__ __attribute__((aligned(16))) float part[kDdThreads * 4];
  const int h = blockIdx.x, b = blockIdx.y, tid = threadIdx.x;
  const int R = a.H / a.G, gh = h / R;
  const int pos = a.row_pos[b], slot = a.row_slot[b];
  const int C = delta_channels(a);
  const int e4 = a.EP >> 2, ng = kDdThreads / e4;  // column pieces, row groups
  const int cg = tid % e4, rg = tid / e4, c = 4 * cg;
  const bool live = rg < ng;
  float* st = a.state + slot * a.s_slot + (long long)h * a.dim * a.EP;
  // the state first: its loads cover the convolution
  float4 S[RPT];
#pragma unroll
  for (int i = 0; i < RPT; ++i) {
    const int r = rg + ng * i;
    S[i] = live && r < a.dim && pos > 0
               ? *reinterpret_cast<const float4*>(st + (long long)r * a.EP + c)
               : make_float4(0.f, 0.f, 0.f, 0.f);
  }
  const float* pj = reinterpret_cast<const float*>(a.proj) + (long long)b * a.ldp;
  float* ring = a.ring + slot * a.r_slot;
  const int nch = 2 * a.dim + a.vdim;
  const bool own_qk = h % R == 0;
  for (int x = tid; x < nch; x += kDdThreads) {
    const bool isv = x >= 2 * a.dim;
    const int ch = isv ? 2 * a.G * a.dim + h * a.vdim + x - 2 * a.dim
                       : x < a.dim ? gh * a.dim + x : (a.G + gh) * a.dim + x - a.dim;
    const float cur = pj[ch];
    float y = a.conv[(long long)(a.taps - 1) * C + ch] * cur;
    for (int j = 1; j < a.taps && j <= pos; ++j)
      y = fmaf(a.conv[(long long)(a.taps - 1 - j) * C + ch],
               ring[(long long)((pos - j) % a.taps) * C + ch], y);
    y = silu32(y);
    if (isv) v[x - 2 * a.dim] = y;
    else if (x < a.dim) q[x] = y;
    else k[x - a.dim] = y;
    if (isv || own_qk) ring[(long long)(pos % a.taps) * C + ch] = cur;
  }
  __syncthreads();
  {  // unit norms: wave 0 the query, wave 1 the key
    const int w = tid >> 6, lane = tid & 63;
    if (w < 2) {
      const float* x = w == 0 ? q : k;
      float ss = 0.f;
      for (int d = lane; d < a.dim; d += 64) ss += x[d] * x[d];
      ss = wave_sum(ss);
      if (lane == 0)
        sn[w] = 1.f / sqrtf(ss + 1e-6f) / (w == 0 ? sqrtf((float)a.dim) : 1.f);
    }
  }
  __syncthreads();
  const float rq = sn[0], rk = sn[1];
  const float* ab = a.ab + (long long)b * a.ldab;
  const float dec = expf(-expf(a.a_log[h]) * softplus32(ab[h] + a.dt_bias[h]));
  const float beta = sigmoid32(ab[a.H + h]);
  float4 acc = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
  for (int i = 0; i < RPT; ++i) {
    const int r = rg + ng * i;
    const float kr = live && r < a.dim ? k[r] * rk : 0.f;
    S[i].x *= dec; S[i].y *= dec; S[i].z *= dec; S[i].w *= dec;
    acc.x = fmaf(kr, S[i].x, acc.x); acc.y = fmaf(kr, S[i].y, acc.y);
    acc.z = fmaf(kr, S[i].z, acc.z); acc.w = fmaf(kr, S[i].w, acc.w);
  }
  if (live) *reinterpret_cast<float4*>(part + rg * a.EP + c) = acc;
  __syncthreads();
  for (int d = tid; d < a.vdim; d += kDdThreads) {
    float s = 0.f;
    for (int g = 0; g < ng; ++g) s += part[g * a.EP + d];
    u[d] = beta * (v[d] - s);
  }
  __syncthreads();
  float uv[4];
#pragma unroll
  for (int e = 0; e < 4; ++e) uv[e] = c + e < a.vdim ? u[c + e] : 0.f;
  acc = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
  for (int i = 0; i < RPT; ++i) {
    const int r = rg + ng * i;
    if (live && r < a.dim) {
      const float kr = k[r] * rk, qr = q[r] * rq;
      S[i].x = fmaf(kr, uv[0], S[i].x); S[i].y = fmaf(kr, uv[1], S[i].y);
      S[i].z = fmaf(kr, uv[2], S[i].z); S[i].w = fmaf(kr, uv[3], S[i].w);
      *reinterpret_cast<float4*>(st + (long long)r * a.EP + c) = S[i];
      acc.x = fmaf(qr, S[i].x, acc.x); acc.y = fmaf(qr, S[i].y, acc.y);
      acc.z = fmaf(qr, S[i].z, acc.z); acc.w = fmaf(qr, S[i].w, acc.w);
    }
  }
  if (live) *reinterpret_cast<float4*>(part + rg * a.EP + c) = acc;
  __syncthreads();
  float ov = 0.f;  // vdim <= 256 < threads
  if (tid < a.vdim)
    for (int g = 0; g < ng; ++g) ov += part[g * a.EP + tid];
  const float rms = 1.f / sqrtf(block_sum(ov * ov, red) / (float)a.vdim + a.eps);
  if (tid < a.vdim)
    reinterpret_cast<E*>(a.out)[(long long)b * a.ldo + h * a.vdim + tid] =
        St<DT>::st(ov * rms * a.norm_w[tid] * silu32(pj[C + h * a.vdim + tid]));
}

}  // namespace cake

using namespace cake;

static bool delta_shape_ok(int H, int G, int dim, int vdim, int EP, int taps) {
  return H > 0 && G > 0 && H % G == 0 && dim > 0 && dim <= 256 && vdim > 0 && vdim <= 256 &&
         EP >= vdim && EP % 4 == 0 && EP <= 256 && taps >= 1;
}

CAKE_API int cake_mixer_delta_prefill(int dt, const void* proj, long long ldp, const float* ab,
                                      long long ldab, int N, int H, int G, int dim, int vdim,
                                      int EP, int taps, float eps, const float* conv,
                                      const float* a_log, const float* dt_bias,
                                      const float* norm_w, float* qn, float* kn, float* vv,
                                      float* tp, float* gm, float* o, float* state, float* ring,
                                      long long s_slot, long long r_slot, const int* row_pos,
                                      const int* row_slot, const int* row_seq0, const void* seq,
                                      int B, const void* chunk, const int* chunk0, int NC,
                                      void* out, long long ldo, hipStream_t st) {
  if (!delta_shape_ok(H, G, dim, vdim, EP, taps) || N <= 0 || B <= 0 || NC < B)
    return (int)hipErrorInvalidValue;
  const int ni = (dim + 63) / 64;
  DeltaArgs a{proj, ldp, ab, ldab, N, H, G, dim, vdim, EP, taps, eps, conv, a_log, dt_bias,
              norm_w, 64 * ni, qn, kn, vv, tp, gm, o, state, ring, s_slot, r_slot, row_pos,
              row_slot, row_seq0, (const SeqRow*)seq, (const int2*)chunk, chunk0, NC, out, ldo};
  const dim3 gp((unsigned)(((long long)NC * (2 * G + H) + 3) / 4));
  const dim3 gs(H, (vdim + 15) / 16, B);
  const dim3 go((unsigned)(((long long)N * H + 3) / 4));
  const int widest = 64 * ni > vdim ? 64 * ni : vdim;
  const int vec = dim % 2 == 0 && vdim % 2 == 0 && ldp % 2 == 0 && ((uintptr_t)proj % 4) == 0;
#define CAKE_PREP1(CPL, W) \
  hipLaunchKernelGGL((mixer_delta_prep_kernel<DT, CPL, W>), gp, dim3(256), 0, st, a, vec)
#define CAKE_PREP(W)                        \
  do {                                      \
    if (widest <= 64) CAKE_PREP1(1, W);     \
    else if (widest <= 128) CAKE_PREP1(2, W); \
    else CAKE_PREP1(4, W);                  \
  } while (0)
  CAKE_MIX_DT(dt, {
    if (taps <= 4) CAKE_PREP(4); else CAKE_PREP(8);
    hipLaunchKernelGGL(mixer_delta_chunk_kernel, dim3((unsigned)(((long long)NC * G + 3) / 4)),
                       dim3(256), 0, st, a);
    if (ni == 1) hipLaunchKernelGGL((mixer_delta_scan_kernel<DT, 1>), gs, dim3(256), 0, st, a);
    else if (ni == 2) hipLaunchKernelGGL((mixer_delta_scan_kernel<DT, 2>), gs, dim3(256), 0, st, a);
    else if (ni == 3) hipLaunchKernelGGL((mixer_delta_scan_kernel<DT, 3>), gs, dim3(256), 0, st, a);
    else hipLaunchKernelGGL((mixer_delta_scan_kernel<DT, 4>), gs, dim3(256), 0, st, a);
    hipLaunchKernelGGL((mixer_delta_out_kernel<DT>), go, dim3(256), 0, st, a);
  });
  return (int)hipGetLastError();
}

CAKE_API int cake_mixer_delta_decode(int dt, const float* proj, long long ldp, const float* ab,
                                     long long ldab, int B, int H, int G, int dim, int vdim, int EP,
                                     int taps, float eps, const float* conv, const float* a_log,
                                     const float* dt_bias, const float* norm_w, float* state,
                                     float* ring, long long s_slot, long long r_slot,
                                     const int* pos, const int* slot, void* out, long long ldo,
                                     hipStream_t st) {
  if (!delta_shape_ok(H, G, dim, vdim, EP, taps) || B <= 0) return (int)hipErrorInvalidValue;
  DeltaArgs a{};
  a.proj = proj; a.ldp = ldp; a.ab = ab; a.ldab = ldab; a.N = B; a.H = H; a.G = G; a.dim = dim;
  a.vdim = vdim; a.EP = EP; a.taps = taps; a.eps = eps; a.conv = conv; a.a_log = a_log;
  a.dt_bias = dt_bias; a.norm_w = norm_w; a.state = state; a.ring = ring; a.s_slot = s_slot;
  a.r_slot = r_slot; a.row_pos = pos; a.row_slot = slot; a.out = out; a.ldo = ldo;
  const int ng = kDdThreads / (EP / 4), rpt = (dim + ng - 1) / ng;
  const dim3 grid(H, B);
#define CAKE_DD(P) hipLaunchKernelGGL((mixer_delta_decode_kernel<DT, P>), grid, dim3(kDdThreads), 0, st, a)
  CAKE_MIX_DT(dt, {
    if (rpt <= 4) CAKE_DD(4);
    else if (rpt <= 8) CAKE_DD(8);
    else if (rpt <= 16) CAKE_DD(16);
    else if (rpt <= 32) CAKE_DD(32);
    else return (int)hipErrorInvalidValue;
  });
#undef CAKE_DD
  return (int)hipGetLastError();
}
