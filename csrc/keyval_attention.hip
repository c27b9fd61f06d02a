// Grouped-query attention over cached rows that are key and value at once,
// bf16, gfx950 matrix cores: position j of KV head g has one row r_j of D
// entries (the key as projected) and one fp32 number f_j (one over its root
// mean square), and
//   score_ij = scale f_j (q_i . r_j) - slope_h (i - j),   o_i = sum_j p_ij r_j
// over the trailing window (or everything), with an optional sink score in the
// denominator. The norm of a key is thus never rounded, and a tile of rows is
// read from memory and staged in LDS ONCE for both products: S^T = R Q^T takes
// its rows, O^T = R^T P^T takes them through ds_read_b64_tr_b16 (a 16-lane
// group reads 4 rows x 16 columns, a lane gets the 4 rows of its column).
//
//   prompt kernel   4 waves; a workgroup owns 128 (token, head) rows of one KV
//                   head: all its query heads of 128 / heads consecutive batch
//                   rows, a wave 32 of them, so the heads of a group share
//                   every staged tile. Queries stay in registers, 64 rows are
//                   staged at a time in one of two LDS buffers, the next ones
//                   are on their way from memory during the products and go
//                   to the other buffer: one barrier per tile.
//                   v_mfma_f32_32x32x16_bf16.
//   token kernel    one (token, KV head, share of the rows) per workgroup,
//                   and every wave on its own: 32 rows at a time into a
//                   private piece of LDS, no workgroup barrier before the
//                   final merge of the four waves. v_mfma_f32_16x16x32_bf16
//                   with up to 16 query heads as the narrow side.
//
// Tiles are walked from the nearest to the farthest: with a distance penalty the
// running maximum then settles in the first tile or two. Where the caller knows
// a bound B of |scale f_j q_i . r_j| (unit-rms queries and keys: scale D), keys
// so far away that B - slope_h distance lies 40 powers of two below -B, the
// least score of the query's own key, are not visited at all: their weights are
// below 2^-40 of the largest one, far less than the rounding of the sum.
//
// In both, the rows of a score tile are read from LDS in an order that leaves
// every lane with runs of 8 consecutive keys of one (token, head): the softmax
// is lane-local plus exchanges between the lanes of one head, and the weights
// pack straight into the operand of the second product as three bf16 terms
// (exact split of the 24-bit mantissa, fp32 accumulation).
#include "mix_common.h"

typedef __attribute__((ext_vector_type(8))) __bf16 kv_bf16x8;
typedef __attribute__((ext_vector_type(16))) float kv_f32x16;
typedef __attribute__((ext_vector_type(4))) float kv_f32x4;
typedef __attribute__((ext_vector_type(4))) short kv_s4;
typedef __attribute__((ext_vector_type(4))) unsigned int kv_u4;
typedef __attribute__((address_space(3))) kv_s4 kv_lds_s4;

#define KV_LOG2E 1.44269504f
#define KV_LOW (-3.0e38f)

union KvPack {
  kv_bf16x8 v;
  kv_s4 h[2];
  unsigned int w[4];
  uint4 q;
};

struct KvArgs {
  unsigned short* out;
  int ldout;
  const unsigned short* q;
  int ldq;
  const unsigned short* rows;   // [NB, G, BS, D]
  const float* kscale;          // [NB, G, BS], or nullptr (1)
  const int* block_tables;
  int max_blocks;
  const int* token_seq;
  const int* token_pos;
  int T, H, G, D, BS;
  float scale2;                 // score scale times log2(e)
  int window, sink;
  const float* sink_vals;       // per head (nullptr: score 0)
  const float* slopes;          // per head (nullptr: no distance term)
  float bound2;                 // bound of the scores times log2(e), < 0: none
  int KS;                       // shares (token kernel)
  float* part;
  int hpb, hblocks;             // heads per workgroup, head blocks per KV head
};

// Two weights (the first one low) cut into three bf16 terms of 8 mantissa bits
// each (truncation; both remainders are exact).
PS_DEV void kv_split(float p0, float p1, unsigned int* a, unsigned int* b,
                     unsigned int* c) {
  const unsigned int x0 = __float_as_uint(p0) & 0xffff0000u;
  const unsigned int x1 = __float_as_uint(p1) & 0xffff0000u;
  const float r0 = p0 - __uint_as_float(x0), r1 = p1 - __uint_as_float(x1);
  const unsigned int y0 = __float_as_uint(r0) & 0xffff0000u;
  const unsigned int y1 = __float_as_uint(r1) & 0xffff0000u;
  const unsigned int z0 = __float_as_uint(r0 - __uint_as_float(y0));
  const unsigned int z1 = __float_as_uint(r1 - __uint_as_float(y1));
  *a = __builtin_amdgcn_perm(x1, x0, 0x07060302u);
  *b = __builtin_amdgcn_perm(y1, y0, 0x07060302u);
  *c = __builtin_amdgcn_perm(z1, z0, 0x07060302u);
}

// Distance from which on no head of h0 .. h0 + n - 1 sees anything that counts
// (see above); a large number where there is no such distance.
PS_DEV int kv_reach(const KvArgs& a, int h0, int n) {
  const int far = 1 << 30;
  if (a.slopes == nullptr || a.bound2 < 0.f) return far;
  float sl = a.slopes[h0];
  for (int h = 1; h < n; ++h) sl = fminf(sl, a.slopes[h0 + h]);
  if (!(sl > 0.f)) return far;
  const float d = (2.0f * a.bound2 + 40.0f) / (sl * KV_LOG2E);
  return d < 1.0e9f ? (int)d + 2 : far;
}

// One online-softmax step of a lane's N scores v (relative to the running
// maximum m, or absolute while m is KV_LOW): weights into v, their sum into l,
// the new maximum into m; returns the factor for what was accumulated before.
// mx: the largest v over all lanes of the row. The factor is 1 for every lane
// (and *moved false) when no maximum of the wave moves.
template <int N>
PS_DEV float kv_softmax(float* v, float mx, float* m, float* l, bool* moved) {
  const bool fresh = *m == KV_LOW;
  *moved = __any(mx > 0.f || (fresh && mx > -INFINITY));
  float alpha = 1.f;
  if (*moved) {
    const float d = fresh ? (mx > -INFINITY ? mx : 0.f) : fmaxf(mx, 0.f);
    if (!fresh) {
      alpha = __builtin_amdgcn_exp2f(-d);
      *m += d;
    } else if (mx > -INFINITY) {
      *m = d;
    }
#pragma unroll
    for (int i = 0; i < N; ++i) v[i] -= d;
  }
  float s = 0.f;
#pragma unroll
  for (int i = 0; i < N; ++i) {
    v[i] = __builtin_amdgcn_exp2f(v[i]);
    s += v[i];
  }
  *l = *l * alpha + s;
  return alpha;
}

// ---------------------------------------------------------------------------
// prompt portions
// ---------------------------------------------------------------------------
#define KV_KT 64

// DK: 16-entry steps of a row (D <= 16 DK; DK even).
template <int DK, int OCC>
__global__ __launch_bounds__(256, OCC) void keyval_prompt_kernel(KvArgs a) {
  constexpr int PK = DK * 16 + 8;
  constexpr int CB = DK / 2;        // 32-column blocks of the output
  __shared__ __align__(16) unsigned short sR[2][KV_KT * PK];
  __shared__ __align__(16) float s_f[2][KV_KT];
  __shared__ int s_row[2][KV_KT];
  __shared__ int s_seq[128], s_pos[128];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int row = lane & 31, hi = lane >> 5;
  const int D = a.D, rep = a.H / a.G, HPB = a.hpb;
  const int TPT = 128 / HPB;
  const int NT = (a.T + TPT - 1) / TPT;

  // heavy workgroups first: later tiles, and the heads with the flattest
  // slopes (the last ones of the usual geometric series)
  const int GH = a.G * a.hblocks;
  const int gh = GH - 1 - blockIdx.x / NT;
  const int tile = NT - 1 - blockIdx.x % NT;
  const int g = gh / a.hblocks, hb = gh % a.hblocks;
  const int tok0 = tile * TPT, ntok = min(TPT, a.T - tok0);
  for (int c = tid; c < ntok; c += 256) {
    s_seq[c] = a.token_seq[tok0 + c];
    s_pos[c] = a.token_pos[tok0 + c];
  }
  __syncthreads();

  // this lane's (token, head)
  const int my = wave * 32 + row;
  const int my_i = my / HPB, my_h = hb * HPB + my % HPB;
  const bool valid = my_i < ntok && my_h < rep;
  const int head = g * rep + min(my_h, rep - 1);
  const int tok = tok0 + min(my_i, ntok - 1);
  const int my_pos = s_pos[min(my_i, ntok - 1)];
  const float sl2 =
      a.slopes != nullptr ? a.slopes[head] * KV_LOG2E : 0.f;
  const int reach =
      kv_reach(a, g * rep + hb * HPB, min(HPB, rep - hb * HPB));
  const int span = a.window > 0 ? min(a.window, reach) : reach;
  // queries: B operand, lane (row, hi) holds entries 16 s + 8 hi + i
  kv_bf16x8 qr[DK];
  {
    const unsigned short* qp = a.q + (size_t)tok * a.ldq + (size_t)head * D;
#pragma unroll
    for (int s = 0; s < DK; ++s) {
      const int c = 16 * s + 8 * hi;
      KvPack u;
      u.q = c < D ? *(const uint4*)(qp + c) : make_uint4(0, 0, 0, 0);
      qr[s] = u.v;
    }
  }
  float m = KV_LOW, l = 0.f;
  if (a.sink) {
    m = (a.sink_vals != nullptr ? a.sink_vals[head] : 0.f) * KV_LOG2E;
    l = hi == 0 ? 1.f : 0.f;  // a row's two lanes are added at the end
  }
  kv_f32x16 acc[CB];
#pragma unroll
  for (int c = 0; c < CB; ++c)
#pragma unroll
    for (int r = 0; r < 16; ++r) acc[c][r] = 0.f;

  constexpr int CPR = DK * 2;                  // 16-byte pieces per row
  constexpr int NP = KV_KT * CPR / 256;        // per thread
  kv_u4 pre[NP];
  float fpre = 0.f;
  // LDS row of this lane's key in a 32-key score tile
  const int krow = (row & 0x13) | ((row & 4) << 1) | ((row & 8) >> 1);
  const int i16 = lane & 15;
  // this lane's part of a transposed read
  const int vat = (8 * hi + (i16 >> 2)) * PK + 16 * ((lane >> 4) & 1) +
                  4 * (i16 & 3);
  const unsigned vis = a.window > 0 ? a.window : 0x7fffffff;

  int rs = 0;
  while (rs < ntok) {
    // batch rows rs .. re - 1 continue one sequence
    int re = rs + 1;
    while (re < ntok && s_seq[re] == s_seq[rs] && s_pos[re] == s_pos[re - 1] + 1)
      ++re;
    const bool mine = valid && my_i >= rs && my_i < re;
    const bool all_mine = __all(mine);
    const int* table = a.block_tables + (size_t)s_seq[rs] * a.max_blocks;
    const int kmin = max(0, s_pos[rs] - span + 1);
    const int kmax = s_pos[re - 1];
    const int nt = (kmax - kmin) / KV_KT + 1;
    // rows of other runs see nothing of this one
    const int pos = mine ? my_pos : -1;
    // what the wave's rows of the run see: all of [w_full_lo, w_first], some
    // of [w_lo, w_last]
    const int ia = max(wave * 32 / HPB, rs);
    const int ib = min((wave * 32 + 31) / HPB, re - 1);
    const bool live = ia <= ib;
    const int w_first = live ? s_pos[ia] : 0, w_last = live ? s_pos[ib] : 0;
    const int w_lo = a.window > 0 ? max(0, w_first - a.window + 1) : 0;
    const int w_full_lo = a.window > 0 ? max(0, w_last - a.window + 1) : 0;

    // page of row (tid & 63) of a tile; rows past the last key repeat it (they
    // are masked). The page number is loaded well ahead of its use.
    auto key_of = [&](int n) {
      return min(kmin + (nt - 1 - n) * KV_KT + (tid & (KV_KT - 1)), kmax);
    };
    auto put_row = [&](int n, int page, int buf) {
      if (tid < KV_KT)
        s_row[buf][tid] = (page * a.G + g) * a.BS + key_of(n) % a.BS;
    };
    auto fetch = [&](int buf) {
      int ri[NP];
#pragma unroll
      for (int u = 0; u < NP; ++u) ri[u] = s_row[buf][(u * 256 + tid) / CPR];
      const int rf = s_row[buf][tid & (KV_KT - 1)];
#pragma unroll
      for (int u = 0; u < NP; ++u) {
        // columns past the row's end repeat its last piece: finite numbers
        // that meet zero query entries or land in columns never stored
        const int c = min((u * 256 + tid) % CPR * 8, D - 8);
        pre[u] = *(const kv_u4*)(a.rows + (int64_t)ri[u] * D + c);
      }
      fpre = a.kscale != nullptr ? a.kscale[rf] : 1.f;
    };
    put_row(0, table[key_of(0) / a.BS], 1);
    __syncthreads();  // also: the previous run's tiles are fully read
    fetch(1);
    int page = table[key_of(min(1, nt - 1)) / a.BS];
    for (int n = 0; n < nt; ++n) {
      // tile n from registers to its buffer, which tile n - 2 has left; what
      // lies past the last tile repeats it
#pragma unroll
      for (int u = 0; u < NP; ++u) {
        const int idx = u * 256 + tid;
        *(kv_u4*)(&sR[n & 1][idx / CPR * PK + idx % CPR * 8]) = pre[u];
      }
      if (tid < KV_KT) s_f[n & 1][tid] = fpre * a.scale2;
      put_row(min(n + 1, nt - 1), page, n & 1);
      __syncthreads();
      fetch(n & 1);
      page = table[key_of(min(n + 2, nt - 1)) / a.BS];
      const unsigned short* sr = sR[n & 1];
      const float* sf = s_f[n & 1];
      const int j0 = kmin + (nt - 1 - n) * KV_KT;
      if (!live || j0 > w_last || j0 + KV_KT - 1 < w_lo) continue;

      kv_f32x16 st[2];
#pragma unroll
      for (int r = 0; r < 16; ++r) st[0][r] = st[1][r] = 0.f;
#pragma unroll
      for (int s = 0; s < DK; ++s) {
        const unsigned short* ka = sr + krow * PK + 16 * s + 8 * hi;
        const kv_bf16x8 a0 = *(const kv_bf16x8*)ka;
        const kv_bf16x8 a1 = *(const kv_bf16x8*)(ka + 32 * PK);
        st[0] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(a0, qr[s], st[0], 0,
                                                        0, 0);
        st[1] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(a1, qr[s], st[1], 0,
                                                        0, 0);
      }
      // st[h][8 s + i] belongs to key j0 + 32 h + 16 s + 8 hi + i
      const float base =
          sl2 * (float)(j0 + 8 * hi - pos) - (m == KV_LOW ? 0.f : m);
      float w[32];
#pragma unroll
      for (int h = 0; h < 2; ++h)
#pragma unroll
        for (int s = 0; s < 2; ++s) {
          const float4 f0 = *(const float4*)(sf + 32 * h + 16 * s + 8 * hi);
          const float4 f1 =
              *(const float4*)(sf + 32 * h + 16 * s + 8 * hi + 4);
          const float f[8] = {f0.x, f0.y, f0.z, f0.w, f1.x, f1.y, f1.z, f1.w};
#pragma unroll
          for (int i = 0; i < 8; ++i)
            w[16 * h + 8 * s + i] =
                fmaf(st[h][8 * s + i], f[i],
                     fmaf(sl2, (float)(32 * h + 16 * s + i), base));
        }
      const int dist = pos - j0 - 8 * hi;  // of this lane's first key
      if (!all_mine || j0 < w_full_lo || j0 + KV_KT - 1 > w_first) {
#pragma unroll
        for (int h = 0; h < 2; ++h)
#pragma unroll
          for (int r = 0; r < 16; ++r) {
            // a distance below zero (a later key) is a huge unsigned number
            const int d = dist - (32 * h + 16 * (r >> 3) + (r & 7));
            if ((unsigned)d >= vis) w[16 * h + r] = -INFINITY;
          }
      }
      float mx = w[0];
#pragma unroll
      for (int i = 1; i < 32; ++i) mx = fmaxf(mx, w[i]);
      mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
      bool moved;
      const float alpha = kv_softmax<32>(w, mx, &m, &l, &moved);
      if (moved) {
#pragma unroll
        for (int c = 0; c < CB; ++c)
#pragma unroll
          for (int r = 0; r < 16; ++r) acc[c][r] *= alpha;
      }
#pragma unroll
      for (int s = 0; s < 4; ++s) {
        KvPack b0, b1, b2;
#pragma unroll
        for (int i = 0; i < 4; ++i)
          kv_split(w[8 * s + 2 * i], w[8 * s + 2 * i + 1], &b0.w[i],
                   &b1.w[i], &b2.w[i]);
#pragma unroll
        for (int c = 0; c < CB; ++c) {
          KvPack v;
#pragma unroll
          for (int h = 0; h < 2; ++h)
            v.h[h] = __builtin_amdgcn_ds_read_tr16_b64_v4i16(
                (kv_lds_s4*)(sr + vat + (16 * s + 4 * h) * PK + 32 * c));
          acc[c] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(v.v, b0.v, acc[c],
                                                           0, 0, 0);
          acc[c] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(v.v, b1.v, acc[c],
                                                           0, 0, 0);
          acc[c] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(v.v, b2.v, acc[c],
                                                           0, 0, 0);
        }
      }
    }
    rs = re;
  }

  l += __shfl_xor(l, 32, 64);  // a lane summed its own keys
  if (!valid) return;
  const float f = 1.0f / l;
  unsigned short* o = a.out + (size_t)tok * a.ldout + (size_t)head * D;
  const bool vec = ((D | a.ldout) & 3) == 0 && ((size_t)a.out & 7) == 0;
  // acc[c][4 q + i] = O[row][32 c + 8 q + 4 hi + i]
#pragma unroll
  for (int c = 0; c < CB; ++c)
#pragma unroll
    for (int q = 0; q < 4; ++q) {
      const int col = 32 * c + 8 * q + 4 * hi;
      unsigned short e[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) e[i] = ps_f32_to_bf16(acc[c][4 * q + i] * f);
      if (vec) {
        if (col < D)
          *(uint2*)(o + col) =
              make_uint2((unsigned int)e[0] | ((unsigned int)e[1] << 16),
                         (unsigned int)e[2] | ((unsigned int)e[3] << 16));
      } else {
#pragma unroll
        for (int i = 0; i < 4; ++i)
          if (col + i < D) o[col + i] = e[i];
      }
    }
}

// ---------------------------------------------------------------------------
// single tokens
// ---------------------------------------------------------------------------
#define KV_TT 32      // rows per tile of a wave
#define KV_HEAD 4     // leading entries of a partial record

// LDS written by some lanes of a wave is read by others of the same wave: the
// wave's LDS accesses complete in order, this keeps the compiler to it.
PS_DEV void kv_wave_sync() {
  __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
  __builtin_amdgcn_wave_barrier();
}

// DK: 32-entry steps of a row (D <= 32 DK).
template <int DK>
__global__ __launch_bounds__(256, DK < 4 ? 4 : DK == 4 ? 3 : 1) void keyval_token_kernel(
    KvArgs a) {
  constexpr int PK = DK * 32 + 8;   // LDS pitch of a row
  constexpr int PA = DK * 32 + 4;   // and of an output row in the merge
  constexpr int NB = DK * 2;        // 16-column blocks of the output
  static_assert(16 * PA * 4 <= KV_TT * PK * 2, "merge fits the row tile");
  __shared__ __align__(16) unsigned short sR[4][KV_TT * PK];
  __shared__ __align__(16) float s_f[4][KV_TT];
  __shared__ float s_m[4][16], s_l[4][16];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int t = blockIdx.x, ks = blockIdx.z;
  const int gh = gridDim.y - 1 - blockIdx.y;  // flattest slopes first
  const int g = gh / a.hblocks, hb = gh % a.hblocks;
  const int D = a.D, rep = a.H / a.G;
  const int nh = min(16, rep - hb * 16);      // heads of this workgroup
  const int h0 = g * rep + hb * 16;
  const int pos = a.token_pos[t];
  const int* table = a.block_tables + (size_t)a.token_seq[t] * a.max_blocks;
  const int reach = kv_reach(a, h0, nh);
  const int lo =
      max(0, pos - (a.window > 0 ? min(a.window, reach) : reach) + 1);
  const int nt = (pos - lo) / KV_TT + 1;
  const int hr = lane & 15, kq = lane >> 4;   // head row, key group
  const int head = h0 + min(hr, nh - 1);
  const float sl2 =
      a.slopes != nullptr ? a.slopes[head] * KV_LOG2E : 0.f;
  unsigned short* sw = sR[wave];
  float* sf = s_f[wave];

  // queries: B operand, lane (hr, kq) holds entries 32 s + 8 kq + i
  kv_bf16x8 qr[DK];
  {
    const unsigned short* qp = a.q + (size_t)t * a.ldq + (size_t)head * D;
#pragma unroll
    for (int s = 0; s < DK; ++s) {
      const int c = 32 * s + 8 * kq;
      KvPack u;
      u.q = c < D ? *(const uint4*)(qp + c) : make_uint4(0, 0, 0, 0);
      qr[s] = u.v;
    }
  }
  // the sink belongs to the first wave of share 0
  float m = KV_LOW, l = 0.f;
  if (a.sink && ks == 0 && wave == 0) {
    m = (a.sink_vals != nullptr ? a.sink_vals[head] : 0.f) * KV_LOG2E;
    l = kq == 0 ? 1.f : 0.f;  // a head's four lanes are added at the end
  }
  kv_f32x4 acc[NB];
#pragma unroll
  for (int c = 0; c < NB; ++c) acc[c] = {0.f, 0.f, 0.f, 0.f};

  constexpr int CPR = DK * 4;               // 16-byte pieces per row
  constexpr int NP = KV_TT * CPR / 64;      // per lane
  uint4 pre[NP];
  float fpre = 1.f;
  // tile n ends at position pos - 32 n; the last one may begin before lo, whose
  // rows it repeats
  auto find = [&](int n) -> int {
    const int j = max(pos - (n + 1) * KV_TT + 1 + (lane & 31), lo);
    return (table[j / a.BS] * a.G + g) * a.BS + (j % a.BS);
  };
  auto fetch = [&](int rowi) {
#pragma unroll
    for (int u = 0; u < NP; ++u) {
      const int idx = u * 64 + lane;
      const int r = idx / CPR, c = (idx - r * CPR) * 8;
      const int ri = __shfl(rowi, r, 64);
      pre[u] = c < D ? *(const uint4*)(a.rows + (int64_t)ri * D + c)
                     : make_uint4(0, 0, 0, 0);
    }
    if (a.kscale != nullptr) fpre = a.kscale[rowi];
  };
  const int step = 4 * a.KS;
  int n = ks * 4 + wave, ahead = 0;
  if (n < nt) {
    fetch(find(n));
    if (n + step < nt) ahead = find(n + step);
  }
  const unsigned short* ka = sw + (8 * (hr >> 2) + (hr & 3)) * PK + 8 * kq;
  const unsigned short* va = sw + (8 * kq + (hr >> 2)) * PK + 4 * (hr & 3);
  for (; n < nt; n += step) {
    kv_wave_sync();  // the previous tile is fully read
#pragma unroll
    for (int u = 0; u < NP; ++u) {
      const int idx = u * 64 + lane;
      const int r = idx / CPR, c = (idx - r * CPR) * 8;
      *(uint4*)(sw + r * PK + c) = pre[u];
    }
    if (lane < KV_TT) sf[lane] = fpre * a.scale2;
    kv_wave_sync();
    if (n + step < nt) {
      fetch(ahead);
      if (n + 2 * step < nt) ahead = find(n + 2 * step);
    }
    // score tile x holds keys 8 (row >> 2) + 4 x + (row & 3): a lane's four
    // entries of both are keys 8 kq .. 8 kq + 7
    kv_f32x4 st[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};
#pragma unroll
    for (int s = 0; s < DK; ++s)
#pragma unroll
      for (int x = 0; x < 2; ++x)
        st[x] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
            *(const kv_bf16x8*)(ka + 4 * x * PK + 32 * s), qr[s], st[x], 0, 0,
            0);
    const int j0 = pos - (n + 1) * KV_TT + 1 + 8 * kq;
    const float base = sl2 * (float)(j0 - pos) - (m == KV_LOW ? 0.f : m);
    float p[8], mx = -INFINITY;
#pragma unroll
    for (int x = 0; x < 2; ++x) {
      const float4 f4 = *(const float4*)(sf + 8 * kq + 4 * x);
      const float f[4] = {f4.x, f4.y, f4.z, f4.w};
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int i = 4 * x + r;
        p[i] = fmaf(st[x][r], f[r], fmaf(sl2, (float)i, base));
        if (j0 + i < lo) p[i] = -INFINITY;
        mx = fmaxf(mx, p[i]);
      }
    }
    mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
    mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
    bool moved;
    const float alpha = kv_softmax<8>(p, mx, &m, &l, &moved);
    if (moved) {
#pragma unroll
      for (int c = 0; c < NB; ++c)
#pragma unroll
        for (int r = 0; r < 4; ++r) acc[c][r] *= alpha;
    }
    KvPack b0, b1, b2;
#pragma unroll
    for (int i = 0; i < 4; ++i)
      kv_split(p[2 * i], p[2 * i + 1], &b0.w[i], &b1.w[i], &b2.w[i]);
#pragma unroll
    for (int c = 0; c < NB; ++c) {
      KvPack v;
#pragma unroll
      for (int h = 0; h < 2; ++h)
        v.h[h] = __builtin_amdgcn_ds_read_tr16_b64_v4i16(
            (kv_lds_s4*)(va + 4 * h * PK + 16 * c));
      acc[c] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(v.v, b0.v, acc[c], 0, 0,
                                                       0);
      acc[c] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(v.v, b1.v, acc[c], 0, 0,
                                                       0);
      acc[c] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(v.v, b2.v, acc[c], 0, 0,
                                                       0);
    }
  }

  // merge of the four waves
  l += __shfl_xor(l, 16, 64);
  l += __shfl_xor(l, 32, 64);
  if (lane < 16) {
    s_m[wave][lane] = m;
    s_l[wave][lane] = l;
  }
  kv_wave_sync();  // the wave's last tile is fully read
  // acc[c][r] = O[head row hr][16 c + 4 kq + r]
  float* sa = (float*)sw + hr * PA + 4 * kq;
#pragma unroll
  for (int c = 0; c < NB; ++c)
    *(float4*)(sa + 16 * c) =
        make_float4(acc[c][0], acc[c][1], acc[c][2], acc[c][3]);
  __syncthreads();
  const int vpr = D / 4;                    // D is a multiple of 8
  const bool vec = (a.ldout & 3) == 0 && ((size_t)a.out & 7) == 0;
  for (int idx = tid; idx < nh * vpr; idx += 256) {
    const int h = idx / vpr, c = (idx - h * vpr) * 4;
    const float mh = fmaxf(fmaxf(s_m[0][h], s_m[1][h]),
                           fmaxf(s_m[2][h], s_m[3][h]));
    float lt = 0.f, o[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int w = 0; w < 4; ++w) {
      const float f = __builtin_amdgcn_exp2f(s_m[w][h] - mh);
      const float4 v = *(const float4*)((const float*)sR[w] + h * PA + c);
      lt += s_l[w][h] * f;
      o[0] += v.x * f;
      o[1] += v.y * f;
      o[2] += v.z * f;
      o[3] += v.w * f;
    }
    if (a.KS == 1) {
      const float f = 1.0f / lt;
      unsigned short* dst =
          a.out + (size_t)t * a.ldout + (size_t)(h0 + h) * D + c;
      unsigned short e[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) e[i] = ps_f32_to_bf16(o[i] * f);
      if (vec)
        *(uint2*)dst =
            make_uint2((unsigned int)e[0] | ((unsigned int)e[1] << 16),
                       (unsigned int)e[2] | ((unsigned int)e[3] << 16));
      else
#pragma unroll
        for (int i = 0; i < 4; ++i) dst[i] = e[i];
    } else {
      // partial record per (token, share, head): max (natural log units),
      // denominator, two unused, D sums
      float* rec = a.part + (((size_t)t * a.KS + ks) * a.H + h0 + h) *
                                (size_t)(D + KV_HEAD);
      if (c == 0) {
        rec[0] = lt > 0.f ? mh * 0.69314718f : PS_NEG_INF;
        rec[1] = lt;
      }
      *(float4*)(rec + KV_HEAD + c) = make_float4(o[0], o[1], o[2], o[3]);
    }
  }
}

extern "C" {

void mx_latent_combine(void* out, int ldout, const void* part, int T_, int H,
                       int DV, int KS, void* stream);

// Returns 0 when launched, 1 when the shape is outside these kernels: rows of
// whole 16-byte vectors, up to 256 entries. token: single tokens (every batch
// row on its own), else prompt portions. bound: of the scores' magnitude before
// the distance penalty (0: unknown).
int mx_keyval_attention(void* out, int ldout, const void* q, int ldq,
                        const void* rows, const void* kscale,
                        const void* block_tables, int max_blocks,
                        const void* token_seq, const void* token_pos, int T_,
                        int H, int G, int D, int BS, float scale, int window,
                        int sink, const void* sink_vals, const void* slopes,
                        float bound, int token, int splits, void* scratch, void* stream) {
  if (T_ <= 0) return 0;
  if (G < 1 || H < 1 || H % G || BS < 1 || D < 8 || D % 8 || D > 256 ||
      ldq % 8 || (((size_t)q | (size_t)rows) & 15))
    return 1;
  typedef unsigned short U;
  const int rep = H / G;
  KvArgs a = {(U*)out, ldout, (const U*)q, ldq, (const U*)rows,
              (const float*)kscale, (const int*)block_tables, max_blocks,
              (const int*)token_seq, (const int*)token_pos, T_, H, G, D, BS,
              scale * KV_LOG2E, window, sink, (const float*)sink_vals,
              (const float*)slopes, bound > 0.f ? bound * KV_LOG2E : -1.f, 1,
              nullptr, 0, 0};
  if (!token) {
    a.hpb = rep < 128 ? rep : 128;
    a.hblocks = (rep + a.hpb - 1) / a.hpb;
    const int tpt = 128 / a.hpb;
    const unsigned grid =
        (unsigned)((T_ + tpt - 1) / tpt) * (unsigned)(G * a.hblocks);
#define KV_GO(DK, OCC)                                                    \
  hipLaunchKernelGGL((keyval_prompt_kernel<DK, OCC>), dim3(grid), dim3(256), \
                     0, (hipStream_t)stream, a)
    if (D <= 64)
      KV_GO(4, 2);
    else if (D <= 96)
      KV_GO(6, 2);
    else if (D <= 128)
      KV_GO(8, 2);
    else if (D <= 192)
      KV_GO(12, 1);
    else
      KV_GO(16, 1);
#undef KV_GO
    return 0;
  }
  a.KS = splits > 1 && scratch != nullptr ? splits : 1;
  if (a.KS > 16) return 1;
  a.part = (float*)scratch;
  a.hpb = 16;
  a.hblocks = (rep + 15) / 16;
  dim3 grid(T_, G * a.hblocks, a.KS);
#define KV_GO(DK)                                                          \
  hipLaunchKernelGGL((keyval_token_kernel<DK>), grid, dim3(256), 0,        \
                     (hipStream_t)stream, a)
  if (D <= 64)
    KV_GO(2);
  else if (D <= 96)
    KV_GO(3);
  else if (D <= 128)
    KV_GO(4);
  else
    KV_GO(8);
#undef KV_GO
  if (a.KS > 1)
    mx_latent_combine(out, ldout, scratch, T_, H, D, a.KS, stream);
  return 0;
}

}  // extern "C"
