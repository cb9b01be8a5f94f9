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
//   * mixer_delta_prep (prompt rows): convolution, SiLU, unit norms, q.k, step size, decay.
//   * mixer_delta_scan: the recurrence of one sequence.  The columns of S are independent
//     given k, q, the decay and the step size, so a workgroup takes 16 columns of one head:
//     16 lanes hold one column in registers, dot products are in-row DPP sums, and the
//     read-out uses o = decay (S^T q) + (q.k) u, so both dots run side by side ahead of u.
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
  float* qn;              // [N][G][dim]
  float* kn;              // [N][G][dim]
  float* vv;              // [N][H][vdim]
  float* qk;              // [N][G]
  float* bd;              // [N][H][2] (decay, beta)
  float* o;               // [N][H][vdim]
  float* state;
  float* ring;
  long long s_slot, r_slot;
  const int* row_pos;     // [N]
  const int* row_slot;    // [N]
  const int* row_seq0;    // [N] packed row of the sequence's first token in this step
  const SeqRow* seq;      // [B]
  void* out;              // [N][ldo]
  long long ldo;
};

__device__ __forceinline__ int delta_channels(const DeltaArgs& a) {
  return 2 * a.G * a.dim + a.H * a.vdim;
}

// convolution + SiLU of channel c at packed row n (prompt rows)
template <int DT>
__device__ __forceinline__ float conv_row(const DeltaArgs& a, int n, int pos, int first, int c,
                                          const float* ring, int C) {
  using E = typename St<DT>::E;
  const E* x = reinterpret_cast<const E*>(a.proj) + c;
  float y = 0.f;
  for (int j = 0; j < a.taps; ++j) {  // j tokens back
    const int p = pos - j;
    if (p < 0) break;
    const int src = n - j;
    const float v = src >= first ? St<DT>::ld(x[(long long)src * a.ldp])
                                 : ring[(long long)(p % a.taps) * C + c];
    y = fmaf(a.conv[(long long)(a.taps - 1 - j) * C + c], v, y);
  }
  return silu32(y);
}

// a wave per (row, unit): units [0, G) = the q and k of one head, [G, G + H) = one value head
template <int DT>
__global__ __launch_bounds__(256) void mixer_delta_prep_kernel(DeltaArgs a) {
  const int lane = threadIdx.x & 63;
  const int units = a.G + a.H;
  const long long item = (long long)blockIdx.x * 4 + (threadIdx.x >> 6);
  if (item >= (long long)a.N * units) return;
  const int n = (int)(item / units), u = (int)(item - (long long)n * units);
  const int C = delta_channels(a);
  const int pos = a.row_pos[n], first = a.row_seq0[n];
  const float* ring = a.ring + a.row_slot[n] * a.r_slot;
  if (u < a.G) {
    float q[4], k[4];
    float sq = 0.f, sk = 0.f, qk = 0.f;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int d = lane + 64 * i;
      q[i] = k[i] = 0.f;
      if (d < a.dim) {
        q[i] = conv_row<DT>(a, n, pos, first, u * a.dim + d, ring, C);
        k[i] = conv_row<DT>(a, n, pos, first, (a.G + u) * a.dim + d, ring, C);
      }
      sq += q[i] * q[i];
      sk += k[i] * k[i];
    }
    const float rq = 1.f / sqrtf(wave_sum(sq) + 1e-6f) / sqrtf((float)a.dim);
    const float rk = 1.f / sqrtf(wave_sum(sk) + 1e-6f);
    float* qo = a.qn + ((long long)n * a.G + u) * a.dim;
    float* ko = a.kn + ((long long)n * a.G + u) * a.dim;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int d = lane + 64 * i;
      q[i] *= rq;
      k[i] *= rk;
      qk += q[i] * k[i];
      if (d < a.dim) { qo[d] = q[i]; ko[d] = k[i]; }
    }
    qk = wave_sum(qk);
    if (lane == 0) a.qk[(long long)n * a.G + u] = qk;
  } else {
    const int h = u - a.G;
    for (int d = lane; d < a.vdim; d += 64)
      a.vv[((long long)n * a.H + h) * a.vdim + d] =
          conv_row<DT>(a, n, pos, first, 2 * a.G * a.dim + h * a.vdim + d, ring, C);
    if (lane == 0) {
      const float* ab = a.ab + (long long)n * a.ldab;
      float* bd = a.bd + ((long long)n * a.H + h) * 2;
      bd[0] = expf(-expf(a.a_log[h]) * softplus32(ab[h] + a.dt_bias[h]));
      bd[1] = sigmoid32(ab[a.H + h]);
    }
  }
}

constexpr int kScanTok = 16;  // tokens staged per round

// grid (ceil(vdim / 16), H, B), 256 threads: wave w = columns 4w..4w+3, 16 lanes per column;
// lane lr holds rows 64 i + 4 lr + {0..3}, i < NI (dim <= 64 NI)
template <int DT, int NI>
__global__ __launch_bounds__(256) void mixer_delta_scan_kernel(DeltaArgs a) {
  using E = typename St<DT>::E;
  constexpr int DR = 64 * NI;
  __shared__ __attribute__((aligned(16))) float ks[2][kScanTok][DR], qs[2][kScanTok][DR];
  __shared__ float vs[2][kScanTok][16], sc[2][kScanTok][4];  // sc: decay, beta, q.k
  const SeqRow sq = a.seq[blockIdx.z];
  const int h = blockIdx.y, R = a.H / a.G, gh = h / R, c0 = blockIdx.x * 16;
  const int tid = threadIdx.x, lane = tid & 63, lr = lane & 15;
  const int cl = (tid >> 6) * 4 + (lane >> 4), col = c0 + cl;
  const bool cok = col < a.vdim;
  float* st = a.state + sq.slot * a.s_slot + (long long)h * a.dim * a.EP;
  float S[NI][4];
#pragma unroll
  for (int i = 0; i < NI; ++i)
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int r = 64 * i + 4 * lr + e;
      S[i][e] = sq.pos0 > 0 && cok && r < a.dim ? st[(long long)r * a.EP + col] : 0.f;
    }
  // staging: thread -> (token tid / 16, 16 lanes over the row), pieces in registers
  const int tt = tid >> 4, tl = tid & 15;
  float pk[4 * NI], pq[4 * NI], pv, ps;
  auto gload = [&](int t0) __attribute__((always_inline)) {
    const int t = min(t0 + tt, sq.len - 1);  // rows past the end repeat the last (not used)
    const long long n = sq.row0 + t;
    const float* kp = a.kn + (n * a.G + gh) * a.dim;
    const float* qp = a.qn + (n * a.G + gh) * a.dim;
#pragma unroll
    for (int i = 0; i < 4 * NI; ++i) {
      const int d = tl + 16 * i;
      pk[i] = d < a.dim ? kp[d] : 0.f;
      pq[i] = d < a.dim ? qp[d] : 0.f;
    }
    pv = c0 + tl < a.vdim ? a.vv[(n * a.H + h) * a.vdim + c0 + tl] : 0.f;
    ps = tl < 2 ? a.bd[(n * a.H + h) * 2 + tl] : tl == 2 ? a.qk[n * a.G + gh] : 0.f;
  };
  auto sstore = [&](int buf) __attribute__((always_inline)) {
#pragma unroll
    for (int i = 0; i < 4 * NI; ++i) {
      ks[buf][tt][tl + 16 * i] = pk[i];
      qs[buf][tt][tl + 16 * i] = pq[i];
    }
    vs[buf][tt][tl] = pv;
    if (tl < 4) sc[buf][tt][tl] = ps;
  };
  gload(0);
  sstore(0);
  __syncthreads();
  int buf = 0;
  for (int t0 = 0; t0 < sq.len; t0 += kScanTok) {
    const bool more = t0 + kScanTok < sq.len;
    if (more) gload(t0 + kScanTok);
    const int nt = min(kScanTok, sq.len - t0);
    float oreg = 0.f;
#pragma unroll 4
    for (int t = 0; t < nt; ++t) {
      float4 kv[NI], qv[NI];
#pragma unroll
      for (int i = 0; i < NI; ++i) {
        kv[i] = *reinterpret_cast<const float4*>(&ks[buf][t][64 * i + 4 * lr]);
        qv[i] = *reinterpret_cast<const float4*>(&qs[buf][t][64 * i + 4 * lr]);
      }
      const float dec = sc[buf][t][0], beta = sc[buf][t][1], qk = sc[buf][t][2];
      const float v = vs[buf][t][cl];
      float ka = 0.f, kb = 0.f, qa = 0.f, qb = 0.f;
#pragma unroll
      for (int i = 0; i < NI; ++i) {
        ka = fmaf(kv[i].x, S[i][0], ka); kb = fmaf(kv[i].y, S[i][1], kb);
        qa = fmaf(qv[i].x, S[i][0], qa); qb = fmaf(qv[i].y, S[i][1], qb);
        ka = fmaf(kv[i].z, S[i][2], ka); kb = fmaf(kv[i].w, S[i][3], kb);
        qa = fmaf(qv[i].z, S[i][2], qa); qb = fmaf(qv[i].w, S[i][3], qb);
      }
      const float kS = row16_sum(ka + kb), qS = row16_sum(qa + qb);
      const float u = beta * (v - dec * kS);
#pragma unroll
      for (int i = 0; i < NI; ++i) {
        S[i][0] = fmaf(kv[i].x, u, dec * S[i][0]);
        S[i][1] = fmaf(kv[i].y, u, dec * S[i][1]);
        S[i][2] = fmaf(kv[i].z, u, dec * S[i][2]);
        S[i][3] = fmaf(kv[i].w, u, dec * S[i][3]);
      }
      const float ov = fmaf(dec, qS, qk * u);
      oreg = lr == t ? ov : oreg;  // lane lr keeps token lr of the round
    }
    if (cok && lr < nt)
      a.o[((long long)(sq.row0 + t0 + lr) * a.H + h) * a.vdim + col] = oreg;
    if (more) sstore(buf ^ 1);
    __syncthreads();
    buf ^= 1;
  }
  if (cok)
#pragma unroll
    for (int i = 0; i < NI; ++i)
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int r = 64 * i + 4 * lr + e;
        if (r < a.dim) st[(long long)r * a.EP + col] = S[i][e];
      }
  // the ring entries of the last taps - 1 tokens (every prompt row has been convolved by now)
  if (blockIdx.x != 0) return;
  const int C = delta_channels(a);
  float* ring = a.ring + sq.slot * a.r_slot;
  const int keep = min(a.taps - 1, sq.len);
  const int nq = h % R == 0 ? 2 * a.dim : 0;  // q and k channels: the group's first head
  for (int i = tid; i < keep * (nq + a.vdim); i += 256) {
    const int j = i / (nq + a.vdim), x = i - j * (nq + a.vdim);
    const int c = x < nq ? (x < a.dim ? gh * a.dim + x : (a.G + gh) * a.dim + x - a.dim)
                         : 2 * a.G * a.dim + h * a.vdim + x - nq;
    const int row = sq.len - 1 - j;
    ring[(long long)((sq.pos0 + row) % a.taps) * C + c] =
        St<DT>::ld(reinterpret_cast<const E*>(a.proj)[(long long)(sq.row0 + row) * a.ldp + c]);
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
  float x[4], ss = 0.f;
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int d = lane + 64 * i;
    x[i] = d < a.vdim ? o[d] : 0.f;
    ss += x[i] * x[i];
  }
  const float r = 1.f / sqrtf(wave_sum(ss) / (float)a.vdim + a.eps);
  const E* gp = reinterpret_cast<const E*>(a.proj) + n * a.ldp + delta_channels(a) + h * a.vdim;
  E* out = reinterpret_cast<E*>(a.out) + n * a.ldo + h * a.vdim;
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
                                      float* qk, float* bd, float* o, float* state, float* ring,
                                      long long s_slot, long long r_slot, const int* row_pos,
                                      const int* row_slot, const int* row_seq0, const void* seq,
                                      int B, void* out, long long ldo, hipStream_t st) {
  if (!delta_shape_ok(H, G, dim, vdim, EP, taps) || N <= 0 || B <= 0)
    return (int)hipErrorInvalidValue;
  DeltaArgs a{proj, ldp, ab, ldab, N, H, G, dim, vdim, EP, taps, eps, conv, a_log, dt_bias,
              norm_w, qn, kn, vv, qk, bd, o, state, ring, s_slot, r_slot, row_pos, row_slot,
              row_seq0, (const SeqRow*)seq, out, ldo};
  const dim3 gp((unsigned)(((long long)N * (G + H) + 3) / 4));
  const dim3 gs((vdim + 15) / 16, H, B);
  const dim3 go((unsigned)(((long long)N * H + 3) / 4));
  const int ni = (dim + 63) / 64;
  CAKE_MIX_DT(dt, {
    hipLaunchKernelGGL((mixer_delta_prep_kernel<DT>), gp, dim3(256), 0, st, a);
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
