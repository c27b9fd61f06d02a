// Causal (windowed) attention of prompt portions over expanded keys and
// values, bf16, gfx950 matrix cores: every query head has keys and values of
// its own, laid out for this kernel by the GEMMs that expand them.
//   q  [T, H*D]        queries, a portion's rows are consecutive positions
//   k  [N, H*D]        key rows; a segment's rows start at a multiple of 64
//                      and are zero-filled up to the next one
//   vt [H*DV, N]       values TRANSPOSED (the GEMM computes W_v C^T), so a
//                      matrix-core operand of 8 consecutive keys is one
//                      16-byte read with no transposition anywhere
//   tiles [NT][4]      (first query row, rows <= 128, first key row of the
//                      segment, position of the first query within it)
//
// A workgroup (4 waves) owns one tile and one head, a wave 32 of its rows.
// Both products run swapped on v_mfma_f32_32x32x16_bf16 (S^T = K Q^T,
// O^T = V^T P^T): a lane's accumulator entries belong to one row (lane & 31),
// the online softmax is lane-local plus one exchange with lane ^ 32, and P
// stays in registers. Key row m of a 32-key score tile is read from LDS row
// m with bits 2 and 3 swapped: a lane then owns runs of 8 consecutive keys,
// the same order in which its V^T operand is read. Queries stay in registers
// for the whole tile; 64 keys are staged at a time, the next ones are on
// their way from memory during the products. Tiles that every row of a wave
// sees take no mask code, tiles that none sees are skipped by that wave.
//
// Scores and softmax are fp32; a weight enters P.V as three bf16 terms
// (exact split of the 24-bit mantissa, fp32 accumulation).
#include "mix_common.h"

typedef __attribute__((ext_vector_type(8))) __bf16 xa_bf16x8;
typedef __attribute__((ext_vector_type(16))) float xa_f32x16;

union XaPack {
  xa_bf16x8 v;
  unsigned int w[4];
  uint4 q;
};

struct XaArgs {
  unsigned short* out;
  int ldout;
  const unsigned short* q;
  int ldq;
  const unsigned short* k;
  const unsigned short* vt;
  int N;                      // rows of k, columns of vt
  const int* tiles;
  int NT, H, D, DV;
  float scale2;               // score scale times log2(e)
  int window;                 // 0: none
  int sink;
  const float* sink_vals;     // per head (nullptr: score 0)
  const unsigned short* gate; // [T, H] head gates before the sigmoid, or null
  int ldgate;
};

#define XA_KT 64                 // keys per stage
#define XA_PV (XA_KT + 8)        // LDS pitch of a V^T row

// DK: 16-entry steps of the key dimension (D <= 16 DK), CB: 32-column blocks
// of the values (DV <= 32 CB).
template <int DK, int CB>
__global__ __launch_bounds__(256, 2) void expand_attn_kernel(XaArgs a) {
  constexpr int PK = DK * 16 + 8;
  __shared__ __align__(16) unsigned short sK[XA_KT * PK];
  __shared__ __align__(16) unsigned short sV[CB * 32 * XA_PV];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int row = lane & 31, hi = lane >> 5;

  // one head's tiles on one XCD (workgroups go round the 8 of them)
  int head, tile;
  if (a.H % 8 == 0) {
    const int k8 = blockIdx.x >> 3;
    head = (blockIdx.x & 7) + 8 * (k8 / a.NT);
    tile = k8 % a.NT;
  } else {
    head = blockIdx.x / a.NT;
    tile = blockIdx.x % a.NT;
  }
  const int* ti = a.tiles + 4 * tile;
  const int row0 = ti[0], nrows = ti[1], key0 = ti[2], pos0 = ti[3];
  const int D = a.D, DV = a.DV;

  // queries: B operand, lane (row, hi) holds entries 16 s + 8 hi + i
  const int my = wave * 32 + row;
  xa_bf16x8 qr[DK];
  {
    const unsigned short* qp = a.q +
                               (size_t)(row0 + min(my, nrows - 1)) * a.ldq +
                               (size_t)head * D;
#pragma unroll
    for (int s = 0; s < DK; ++s) {
      const int c = 16 * s + 8 * hi;
      XaPack u;
      u.q = c < D ? *(const uint4*)(qp + c) : make_uint4(0, 0, 0, 0);
      qr[s] = u.v;
    }
  }
  const int pos = pos0 + my;
  const int lo = a.window > 0 ? max(0, pos - a.window + 1) : 0;
  // what the wave's rows see: all of [w_full_lo, w_first], some of
  // [w_lo, w_last]
  const int w_first = pos0 + wave * 32, w_last = w_first + 31;
  const int w_lo = a.window > 0 ? max(0, w_first - a.window + 1) : 0;
  const int w_full_lo = a.window > 0 ? max(0, w_last - a.window + 1) : 0;
  const bool live = wave * 32 < nrows;

  float m = -3.0e38f, l = 0.f;
  if (a.sink) {
    m = (a.sink_vals != nullptr ? a.sink_vals[head] : 0.f) * 1.44269504f;
    l = hi == 0 ? 1.f : 0.f;  // a row's two lanes are added at the end
  }
  xa_f32x16 acc[CB];
#pragma unroll
  for (int c = 0; c < CB; ++c)
#pragma unroll
    for (int r = 0; r < 16; ++r) acc[c][r] = 0.f;

  const int kstart =
      (a.window > 0 ? max(0, pos0 - a.window + 1) : 0) & ~(XA_KT - 1);
  const int klast = pos0 + nrows - 1;
  const size_t ldk = (size_t)a.H * D;
  const unsigned short* kbase = a.k + (size_t)key0 * ldk + (size_t)head * D;
  const unsigned short* vbase = a.vt + (size_t)head * DV * a.N + key0;

  // staging shares: 16-byte pieces of the K and V^T tiles
  constexpr int CPR = DK * 2;                    // pieces per key row
  constexpr int NK = XA_KT * CPR / 256;          // per thread
  constexpr int NV = CB * 32 * (XA_KT / 8) / 256;
  uint4 pk[NK], pv[NV];
  auto fetch = [&](int j0) {
#pragma unroll
    for (int u = 0; u < NK; ++u) {
      const int idx = u * 256 + tid;
      const int r = idx / CPR, c = (idx - r * CPR) * 8;
      pk[u] = c < D ? *(const uint4*)(kbase + (size_t)(j0 + r) * ldk + c)
                    : make_uint4(0, 0, 0, 0);
    }
#pragma unroll
    for (int u = 0; u < NV; ++u) {
      const int idx = u * 256 + tid;
      const int r = idx >> 3, c = (idx & 7) * 8;
      pv[u] = r < DV ? *(const uint4*)(vbase + (size_t)r * a.N + j0 + c)
                     : make_uint4(0, 0, 0, 0);
    }
  };
  fetch(kstart);
  // LDS row of this lane's key in a 32-key score tile
  const int krow = (row & 0x13) | ((row & 4) << 1) | ((row & 8) >> 1);
  for (int j0 = kstart; j0 <= klast; j0 += XA_KT) {
    __syncthreads();  // the previous tile is fully read
#pragma unroll
    for (int u = 0; u < NK; ++u) {
      const int idx = u * 256 + tid;
      const int r = idx / CPR, c = (idx - r * CPR) * 8;
      *(uint4*)(sK + r * PK + c) = pk[u];
    }
#pragma unroll
    for (int u = 0; u < NV; ++u) {
      const int idx = u * 256 + tid;
      *(uint4*)(sV + (idx >> 3) * XA_PV + (idx & 7) * 8) = pv[u];
    }
    __syncthreads();
    if (j0 + XA_KT <= klast) fetch(j0 + XA_KT);
    if (!live || j0 > w_last || j0 + XA_KT - 1 < w_lo) continue;

    xa_f32x16 st[2];
#pragma unroll
    for (int r = 0; r < 16; ++r) st[0][r] = st[1][r] = 0.f;
#pragma unroll
    for (int s = 0; s < DK; ++s) {
      const unsigned short* ka = sK + krow * PK + 16 * s + 8 * hi;
      const xa_bf16x8 a0 = *(const xa_bf16x8*)ka;
      const xa_bf16x8 a1 = *(const xa_bf16x8*)(ka + 32 * PK);
      st[0] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(a0, qr[s], st[0], 0, 0,
                                                      0);
      st[1] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(a1, qr[s], st[1], 0, 0,
                                                      0);
    }
    // st[h][8 s + i] = score of key j0 + 32 h + 16 s + 8 hi + i
    if (j0 < w_full_lo || j0 + XA_KT - 1 > w_first) {
#pragma unroll
      for (int h = 0; h < 2; ++h)
#pragma unroll
        for (int r = 0; r < 16; ++r) {
          const int j = j0 + 32 * h + 16 * (r >> 3) + 8 * hi + (r & 7);
          if (j > pos || j < lo) st[h][r] = -INFINITY;
        }
    }
    float mx = st[0][0];
#pragma unroll
    for (int r = 0; r < 16; ++r) mx = fmaxf(mx, fmaxf(st[0][r], st[1][r]));
    mx = fmaxf(mx, __shfl_xor(mx, 32, 64)) * a.scale2;
    const float mnew = fmaxf(m, mx);
    const float alpha = __builtin_amdgcn_exp2f(m - mnew);
    float ps = 0.f;
#pragma unroll
    for (int h = 0; h < 2; ++h)
#pragma unroll
      for (int r = 0; r < 16; ++r) {
        const float p =
            __builtin_amdgcn_exp2f(fmaf(st[h][r], a.scale2, -mnew));
        st[h][r] = p;
        ps += p;
      }
    l = l * alpha + ps;
    m = mnew;
    if (__any(alpha != 1.f)) {
#pragma unroll
      for (int c = 0; c < CB; ++c)
#pragma unroll
        for (int r = 0; r < 16; ++r) acc[c][r] *= alpha;
    }
#pragma unroll
    for (int s = 0; s < 4; ++s) {
      // p >= 0 cut into three bf16 terms of 8 mantissa bits each
      // (truncation; both remainders are exact)
      XaPack b0, b1, b2;
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        unsigned int h0[2], h1[2], h2[2];
#pragma unroll
        for (int e = 0; e < 2; ++e) {
          const float p = st[s >> 1][8 * (s & 1) + 2 * i + e];
          h0[e] = __float_as_uint(p) & 0xffff0000u;
          const float r1 = p - __uint_as_float(h0[e]);
          h1[e] = __float_as_uint(r1) & 0xffff0000u;
          h2[e] = __float_as_uint(r1 - __uint_as_float(h1[e]));
        }
        // high halves of the pair, the first entry low
        b0.w[i] = __builtin_amdgcn_perm(h0[1], h0[0], 0x07060302u);
        b1.w[i] = __builtin_amdgcn_perm(h1[1], h1[0], 0x07060302u);
        b2.w[i] = __builtin_amdgcn_perm(h2[1], h2[0], 0x07060302u);
      }
#pragma unroll
      for (int c = 0; c < CB; ++c) {
        const xa_bf16x8 v = *(const xa_bf16x8*)(
            sV + (c * 32 + row) * XA_PV + 16 * s + 8 * hi);
        acc[c] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(v, b0.v, acc[c], 0,
                                                         0, 0);
        acc[c] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(v, b1.v, acc[c], 0,
                                                         0, 0);
        acc[c] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(v, b2.v, acc[c], 0,
                                                         0, 0);
      }
    }
  }

  l += __shfl_xor(l, 32, 64);  // a lane summed its own keys
  if (my >= nrows) return;
  float f = 1.0f / l;
  const size_t t = (size_t)row0 + my;
  if (a.gate != nullptr)
    f *= mx_sigmoid(ps_bf16_to_f32(a.gate[t * a.ldgate + head]));
  unsigned short* o = a.out + t * a.ldout + (size_t)head * DV;
  const bool vec = ((DV | a.ldout) & 3) == 0 && ((size_t)a.out & 7) == 0;
  // acc[c][4 g + i] = O[row][32 c + 8 g + 4 hi + i]
#pragma unroll
  for (int c = 0; c < CB; ++c)
#pragma unroll
    for (int g = 0; g < 4; ++g) {
      const int col = 32 * c + 8 * g + 4 * hi;
      unsigned short e[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) e[i] = ps_f32_to_bf16(acc[c][4 * g + i] * f);
      if (vec) {
        if (col < DV)
          *(uint2*)(o + col) =
              make_uint2((unsigned int)e[0] | ((unsigned int)e[1] << 16),
                         (unsigned int)e[2] | ((unsigned int)e[3] << 16));
      } else {
#pragma unroll
        for (int i = 0; i < 4; ++i)
          if (col + i < DV) o[col + i] = e[i];
      }
    }
}

// Returns 0 when launched, 1 when the shape is outside this kernel: head
// widths that are multiples of 8 up to 192 (keys) and any up to 128 (values).
extern "C" int mx_expand_attention(
    void* out, int ldout, const void* q, int ldq, const void* k,
    const void* vt, int N, const void* tiles, int NT, int H, int D, int DV,
    float scale, int window, int sink, const void* sink_vals,
    const void* gate, int ldgate, void* stream) {
  if (NT <= 0) return 0;
  if (D < 8 || D % 8 || D > 192 || DV < 1 || DV > 128 || ldq % 8 || N % 64 ||
      (((size_t)q | (size_t)k | (size_t)vt) & 15))
    return 1;
  typedef unsigned short U;
  const XaArgs a = {(U*)out, ldout, (const U*)q, ldq, (const U*)k,
                    (const U*)vt, N, (const int*)tiles, NT, H, D, DV,
                    scale * 1.44269504f, window, sink,
                    (const float*)sink_vals, (const U*)gate, ldgate};
#define XA_GO(DK, CB)                                                      \
  hipLaunchKernelGGL((expand_attn_kernel<DK, CB>), dim3(NT * H), dim3(256), 0, \
                     (hipStream_t)stream, a)
#define XA_CB(DK)            \
  if (DV <= 64)              \
    XA_GO(DK, 2);            \
  else                       \
    XA_GO(DK, 4)
  if (D <= 64) {
    XA_CB(4);
  } else if (D <= 96) {
    XA_CB(6);
  } else if (D <= 128) {
    XA_CB(8);
  } else {
    XA_CB(12);
  }
#undef XA_CB
#undef XA_GO
  return 0;
}
