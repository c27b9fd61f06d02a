// Single-token attention over latent rows, bf16, gfx950 matrix cores: one
// cached row [latent | rotary key part] per position is key and, in its
// leading DV entries, value of every query head.
//
// A workgroup (8 waves) owns one token, 32 of its heads and one share of its
// keys (shares deal 64-key tiles round-robin and leave partial records that a
// combine pass merges). Per tile:
//   scores   wave (g, rh) forms S^T of 16 keys x 16 heads on
//            v_mfma_f32_16x16x32_bf16; queries stay in registers;
//   softmax  tile maxima of the four key groups meet in LDS, then every lane
//            turns its four scores into weights, stored in LDS as three bf16
//            terms (exact split, fp32 accumulation later);
//   output   wave w owns 32 CW value columns of all 32 heads:
//            O^T += V^T P^T on v_mfma_f32_32x32x16_bf16. The V^T operand
//            comes out of the row-major tile with ds_read_b64_tr_b16 (a
//            16-lane group reads 4 keys x 16 columns, a lane gets the 4 keys
//            of its column).
// No product is computed twice. The next tile is on its way into registers
// while this one is computed, the page-table entries are one tile further
// ahead: a step reads each row once from memory, and hiding that latency is
// what the time depends on.
#include "mix_common.h"

typedef __attribute__((ext_vector_type(8))) __bf16 ld_bf16x8;
typedef __attribute__((ext_vector_type(4))) float ld_f32x4;
typedef __attribute__((ext_vector_type(16))) float ld_f32x16;
typedef __attribute__((ext_vector_type(4))) short ld_s4;
typedef __attribute__((address_space(3))) ld_s4 ld_lds_s4;

#define LD_KT 64         // keys per tile
#define LD_PP (LD_KT + 8)  // LDS pitch of a weight row
#define LD_HEAD 4        // leading entries of a partial record

union LdPack {
  ld_bf16x8 v;
  ld_s4 h[2];
  uint4 q;
};

struct LdArgs {
  unsigned short* out;
  int ldout;
  const unsigned short* q;
  int ldq;
  const unsigned short* cache;  // [NB, 1, BS, D]
  const int* block_tables;
  int max_blocks;
  const int* token_seq;
  const int* token_pos;
  int H, D, DV, BS;
  float scale2;                 // score scale times log2(e)
  int window, sink;
  const float* sink_vals;
  int KS;
  float* part;
};

// DK: 32-entry steps of a row (D <= 32 DK), CW: 32-column blocks per wave
// (DV <= 256 CW).
template <int DK, int CW>
__global__ __launch_bounds__(512, 2) void latent_decode_kernel(LdArgs a) {
  constexpr int PK = DK * 32 + 8;
  __shared__ __align__(16) unsigned short sK[LD_KT * PK];
  __shared__ __align__(16) unsigned short sP[3][32 * LD_PP];
  __shared__ int64_t s_base[2][LD_KT];
  __shared__ float s_max[4][32], s_sum[4][32];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int t = blockIdx.x, ks = blockIdx.z, hb = blockIdx.y * 32;
  const int D = a.D, DV = a.DV;
  const int pos = a.token_pos[t];
  const int* table = a.block_tables + (size_t)a.token_seq[t] * a.max_blocks;
  const int lo = a.window > 0 ? max(0, pos - a.window + 1) : 0;
  const int ntiles = (pos - lo) / LD_KT + 1;

  // scores: this wave's key group and head half
  const int g = wave & 3, rh = wave >> 2;
  const int srow = 16 * rh + (lane & 15);   // head row of the score entries
  const int kq = lane >> 4;
  ld_bf16x8 qr[DK];
  {
    const int head = hb + srow;
    const unsigned short* qp =
        a.q + (size_t)t * a.ldq + (size_t)min(head, a.H - 1) * D;
#pragma unroll
    for (int s = 0; s < DK; ++s) {
      const int c = 32 * s + 8 * kq;
      LdPack u;
      u.q = c < D ? *(const uint4*)(qp + c) : make_uint4(0, 0, 0, 0);
      qr[s] = u.v;
    }
  }
  // output: this wave's columns, all 32 head rows
  const int orow = lane & 31, hi = lane >> 5;
  const int col0 = wave * 32 * CW;
  const bool cols = col0 < DV;
  auto sink2 = [&](int r) -> float {
    return (a.sink_vals != nullptr ? a.sink_vals[min(hb + r, a.H - 1)] : 0.f) *
           1.44269504f;
  };
  const bool own_sink = a.sink && ks == 0;
  float m_s = own_sink ? sink2(srow) : -3.0e38f;   // of head row srow
  float m_o = own_sink ? sink2(orow) : -3.0e38f;   // of head row orow
  float l = 0.f;                                   // this lane's weights
  ld_f32x16 acc[CW];
#pragma unroll
  for (int c = 0; c < CW; ++c)
#pragma unroll
    for (int r = 0; r < 16; ++r) acc[c][r] = 0.f;

  constexpr int CPR = DK * 4;                 // 16-byte pieces per row
  constexpr int NP = LD_KT * CPR / 512;       // per thread
  static_assert(LD_KT * CPR % 512 == 0, "whole pieces per thread");
  uint4 pre[NP];
  auto bases = [&](int tile, int buf) {
    if (tid < LD_KT) {
      // rows past the last key repeat it; they are masked
      const int j = min(lo + tile * LD_KT + tid, pos);
      s_base[buf][tid] =
          ((int64_t)table[j / a.BS] * a.BS + (j % a.BS)) * (int64_t)D;
    }
  };
  auto fetch = [&](int buf) {
#pragma unroll
    for (int u = 0; u < NP; ++u) {
      const int idx = u * 512 + tid;
      const int r = idx / CPR, c = (idx - r * CPR) * 8;
      pre[u] = c < D ? *(const uint4*)(a.cache + s_base[buf][r] + c)
                     : make_uint4(0, 0, 0, 0);
    }
  };
  int tile = ks, it = 0;
  if (tile < ntiles) {
    bases(tile, 0);
    if (tile + a.KS < ntiles) bases(tile + a.KS, 1);
    __syncthreads();
    fetch(0);
  }
  for (; tile < ntiles; tile += a.KS, ++it) {
    __syncthreads();  // the previous tile and its weights are fully read
#pragma unroll
    for (int u = 0; u < NP; ++u) {
      const int idx = u * 512 + tid;
      const int r = idx / CPR, c = (idx - r * CPR) * 8;
      *(uint4*)(sK + r * PK + c) = pre[u];
    }
    // buffer it & 1 held this tile's rows, which are all fetched
    if (tile + 2 * a.KS < ntiles) bases(tile + 2 * a.KS, it & 1);
    __syncthreads();
    if (tile + a.KS < ntiles) fetch((it + 1) & 1);

    const int j0 = lo + tile * LD_KT;
    ld_f32x4 st = {0.f, 0.f, 0.f, 0.f};
    {
      const unsigned short* ka = sK + (16 * g + (lane & 15)) * PK + 8 * kq;
#pragma unroll
      for (int s = 0; s < DK; ++s)
        st = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
            *(const ld_bf16x8*)(ka + 32 * s), qr[s], st, 0, 0, 0);
    }
    // st[r] = score of key j0 + 16 g + 4 kq + r for head row srow
    float mx = -INFINITY;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      if (j0 + 16 * g + 4 * kq + r > pos) st[r] = -INFINITY;
      mx = fmaxf(mx, st[r]);
    }
    mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
    mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
    if (lane < 16) s_max[g][srow] = mx * a.scale2;
    __syncthreads();
    auto tile_max = [&](int r) {
      return fmaxf(fmaxf(s_max[0][r], s_max[1][r]),
                   fmaxf(s_max[2][r], s_max[3][r]));
    };
    {
      const float mnew = fmaxf(m_s, tile_max(srow));
      l *= __builtin_amdgcn_exp2f(m_s - mnew);
      m_s = mnew;
      unsigned int h0[4], h1[4], h2[4];
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const float p =
            __builtin_amdgcn_exp2f(fmaf(st[r], a.scale2, -mnew));
        l += p;
        // three bf16 terms of 8 mantissa bits each (truncation; both
        // remainders are exact)
        h0[r] = __float_as_uint(p) & 0xffff0000u;
        const float r1 = p - __uint_as_float(h0[r]);
        h1[r] = __float_as_uint(r1) & 0xffff0000u;
        h2[r] = __float_as_uint(r1 - __uint_as_float(h1[r]));
      }
      const int at = srow * LD_PP + 16 * g + 4 * kq;
      *(uint2*)(&sP[0][at]) =
          make_uint2(__builtin_amdgcn_perm(h0[1], h0[0], 0x07060302u),
                     __builtin_amdgcn_perm(h0[3], h0[2], 0x07060302u));
      *(uint2*)(&sP[1][at]) =
          make_uint2(__builtin_amdgcn_perm(h1[1], h1[0], 0x07060302u),
                     __builtin_amdgcn_perm(h1[3], h1[2], 0x07060302u));
      *(uint2*)(&sP[2][at]) =
          make_uint2(__builtin_amdgcn_perm(h2[1], h2[0], 0x07060302u),
                     __builtin_amdgcn_perm(h2[3], h2[2], 0x07060302u));
    }
    {
      const float mnew = fmaxf(m_o, tile_max(orow));
      const float alpha = __builtin_amdgcn_exp2f(m_o - mnew);
      m_o = mnew;
      if (__any(alpha != 1.f)) {
#pragma unroll
        for (int c = 0; c < CW; ++c)
#pragma unroll
          for (int r = 0; r < 16; ++r) acc[c][r] *= alpha;
      }
    }
    __syncthreads();
    if (cols) {
      const int i16 = lane & 15;
      // this lane's part of a transposed read: key i16 >> 2 of four, four
      // columns from 16 ((lane >> 4) & 1) + 4 (i16 & 3) on
      const unsigned short* va =
          sK + (8 * hi + (i16 >> 2)) * PK + col0 +
          16 * ((lane >> 4) & 1) + 4 * (i16 & 3);
      const unsigned short* pa = &sP[0][orow * LD_PP + 8 * hi];
#pragma unroll
      for (int s = 0; s < LD_KT / 16; ++s) {
        const ld_bf16x8 b0 = *(const ld_bf16x8*)(pa + 16 * s);
        const ld_bf16x8 b1 = *(const ld_bf16x8*)(pa + 32 * LD_PP + 16 * s);
        const ld_bf16x8 b2 = *(const ld_bf16x8*)(pa + 64 * LD_PP + 16 * s);
#pragma unroll
        for (int c = 0; c < CW; ++c) {
          LdPack v;
#pragma unroll
          for (int h = 0; h < 2; ++h)
            v.h[h] = __builtin_amdgcn_ds_read_tr16_b64_v4i16(
                (ld_lds_s4*)(va + (16 * s + 4 * h) * PK + 32 * c));
          acc[c] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(v.v, b0, acc[c], 0,
                                                           0, 0);
          acc[c] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(v.v, b1, acc[c], 0,
                                                           0, 0);
          acc[c] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(v.v, b2, acc[c], 0,
                                                           0, 0);
        }
      }
    }
  }

  // denominators: lanes of one head row, then the four key groups
  l += __shfl_xor(l, 16, 64);
  l += __shfl_xor(l, 32, 64);
  if (lane < 16) s_sum[g][srow] = l;
  __syncthreads();
  float lt = (s_sum[0][orow] + s_sum[1][orow]) +
             (s_sum[2][orow] + s_sum[3][orow]);
  if (own_sink) lt += __builtin_amdgcn_exp2f(sink2(orow) - m_o);
  const int head = hb + orow;
  if (head >= a.H) return;
  // acc[c][4 q + i] = O[orow][col0 + 32 c + 8 q + 4 hi + i]
  const bool vec = (DV & 3) == 0;
  if (a.KS == 1) {
    const float f = 1.0f / lt;
    unsigned short* o = a.out + (size_t)t * a.ldout + (size_t)head * DV;
    const bool vec2 = vec && (a.ldout & 3) == 0 && ((size_t)a.out & 7) == 0;
#pragma unroll
    for (int c = 0; c < CW; ++c)
#pragma unroll
      for (int q = 0; q < 4; ++q) {
        const int col = col0 + 32 * c + 8 * q + 4 * hi;
        unsigned short e[4];
#pragma unroll
        for (int i = 0; i < 4; ++i)
          e[i] = ps_f32_to_bf16(acc[c][4 * q + i] * f);
        if (vec2) {
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
  } else {
    // partial record per (token, share, head): max (natural log units),
    // denominator, two unused, DV sums
    float* rec = a.part + (((size_t)t * a.KS + ks) * a.H + head) *
                              (size_t)(DV + LD_HEAD);
    if (wave == 0 && hi == 0) {
      rec[0] = lt > 0.f ? m_o * 0.69314718f : PS_NEG_INF;
      rec[1] = lt;
    }
#pragma unroll
    for (int c = 0; c < CW; ++c)
#pragma unroll
      for (int q = 0; q < 4; ++q) {
        const int col = col0 + 32 * c + 8 * q + 4 * hi;
        if (vec) {
          if (col < DV)
            *(float4*)(rec + LD_HEAD + col) =
                make_float4(acc[c][4 * q], acc[c][4 * q + 1],
                            acc[c][4 * q + 2], acc[c][4 * q + 3]);
        } else {
#pragma unroll
          for (int i = 0; i < 4; ++i)
            if (col + i < DV) rec[LD_HEAD + col + i] = acc[c][4 * q + i];
        }
      }
  }
}

// Merge the KS partial records of every (token, head).
__global__ __launch_bounds__(256) void latent_decode_combine_kernel(
    unsigned short* __restrict__ out, int ldout,
    const float* __restrict__ part, int H, int DV, int KS) {
  const int t = blockIdx.x, h = blockIdx.y;
  const float* rec = part + ((size_t)t * KS * H + h) * (DV + LD_HEAD);
  const size_t step = (size_t)H * (DV + LD_HEAD);
  float mh = PS_NEG_INF;
  for (int s = 0; s < KS; ++s) mh = fmaxf(mh, rec[s * step]);
  float w[16], l = 0.f;
#pragma unroll
  for (int s = 0; s < 16; ++s) {
    w[s] = 0.f;
    if (s < KS && rec[s * step] > PS_NEG_INF) {
      w[s] = expf(rec[s * step] - mh);
      l += rec[s * step + 1] * w[s];
    }
  }
  const float inv = 1.0f / l;
  for (int d = threadIdx.x; d < DV; d += blockDim.x) {
    float acc = 0.f;
#pragma unroll
    for (int s = 0; s < 16; ++s)
      if (s < KS && w[s] > 0.f) acc += w[s] * rec[s * step + LD_HEAD + d];
    out[(size_t)t * ldout + h * DV + d] = ps_f32_to_bf16(acc * inv);
  }
}

// Merge pass over partial records as above, at most 16 shares.
extern "C" void mx_latent_combine(void* out, int ldout, const void* part,
                                  int T_, int H, int DV, int KS,
                                  void* stream) {
  hipLaunchKernelGGL(latent_decode_combine_kernel, dim3(T_, H),
                     dim3(DV <= 64 ? 64 : (DV <= 128 ? 128 : 256)), 0,
                     (hipStream_t)stream, (unsigned short*)out, ldout,
                     (const float*)part, H, DV, KS);
}

// Returns 0 when launched, 1 when the shape is outside this kernel: rows of
// whole 16-byte vectors, up to 320 entries with at most 256 value columns or
// up to 576 with at most 512.
extern "C" int mx_latent_decode(
    void* out, int ldout, const void* q, int ldq, const void* cache,
    const void* block_tables, int max_blocks, const void* token_seq,
    const void* token_pos, int T_, int H, int D, int DV, int BS, float scale,
    int window, int sink, const void* sink_vals, int splits, void* scratch,
    void* stream) {
  if (T_ <= 0) return 0;
  if (D % 8 || ldq % 8 || DV < 1 || DV > D || H < 1 || D > 576 || DV > 512 ||
      (((size_t)q | (size_t)cache) & 15))
    return 1;
  const int KS = splits > 1 && scratch != nullptr ? splits : 1;
  if (KS > 16) return 1;
  typedef unsigned short U;
  const LdArgs a = {(U*)out, ldout, (const U*)q, ldq, (const U*)cache,
                    (const int*)block_tables, max_blocks,
                    (const int*)token_seq, (const int*)token_pos, H, D, DV,
                    BS, scale * 1.44269504f, window, sink,
                    (const float*)sink_vals, KS, (float*)scratch};
  dim3 grid(T_, (H + 31) / 32, KS);
#define LD_GO(DK, CW)                                                         \
  hipLaunchKernelGGL((latent_decode_kernel<DK, CW>), grid, dim3(512), 0,      \
                     (hipStream_t)stream, a)
  if (D <= 128 && DV <= 256)
    LD_GO(4, 1);
  else if (D <= 320 && DV <= 256)
    LD_GO(10, 1);
  else
    LD_GO(18, 2);
#undef LD_GO
  if (KS > 1) mx_latent_combine(out, ldout, scratch, T_, H, DV, KS, stream);
  return 0;
}
