// Per-token preparation kernels of the attention and recurrent mixers:
//   attn_prep        per-head query/key RMSNorm, rotary turn of the heads'
//                    leading entries, value blend with another layer's
//                    values, paged K/V append;
//   keyval_prep      queries over their root mean square per head, paged
//                    append of keys that are also the values, with one over
//                    their root mean square beside them;
//   latent_prep      latent RMSNorm, rotary turn of the shared key part and
//                    of the queries' rotary parts, paged append of
//                    [latent | key part], assembly of the latent-space
//                    queries;
//   rms_norm_rows    rows over their root mean square, times a weight (the
//                    latent a query passes);
//   merge_heads      per-head outputs side by side, each head times the
//                    sigmoid of its gate;
//   latent_gather    rows of a paged cache side by side (the rows a step's
//                    prompt portions see, for expansion);
//   pool_append      mean key/value of every block of positions a step
//                    completes, into the pooled caches;
//   short_conv_silu  causal per-channel convolution over time + silu with
//                    the last taps-1 inputs of every sequence as state.
// All arithmetic is fp32; the element type decides loads and the final
// rounding.
#include "mix_common.h"

// One wave per head: x / sqrt(mean(x^2) + eps) * w over D entries (the mean
// over the head, or with ALL over the whole query / key projection, whose
// weights then have H*D / G*D entries), then the first rot_dims entries turn
// by row `position` of the table cs [table_rows][rot_dims / 2][cos, sin].
// Interleaved pairs (2i, 2i+1): a lane reads its own entry and its pair
// partner's (a neighbouring lane's) before it stores, and the wave runs in
// step, so the query is rewritten in place. HALF pairs (i, i + rot_dims / 2):
// a lane owns both entries of a pair, reads them, turns them and stores
// them, so nothing it reads is another lane's to write.
template <typename T, bool HALF, bool ALL>
__global__ __launch_bounds__(256) void attn_prep_kernel(
    T* __restrict__ q, int ldq, const T* __restrict__ k, int ldk,
    T* __restrict__ v, int ldv, const float* __restrict__ qw,
    const float* __restrict__ kw, float eps, const float* __restrict__ vmix,
    const T* __restrict__ vfirst, int ldvf, T* __restrict__ kc,
    T* __restrict__ vc, const int64_t* __restrict__ slots, int H, int G,
    int D, int DV, int BS, const float* __restrict__ cs, int table_rows,
    int rot_dims, const int* __restrict__ positions) {
  __shared__ float red[17];
  const int t = blockIdx.x;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int nw = blockDim.x >> 6;
  const float* csr = nullptr;
  if (cs != nullptr)
    csr = cs + (size_t)min(max(positions[t], 0), table_rows - 1) * rot_dims;
  const int64_t slot = slots[t];
  const int64_t blk = slot >= 0 ? slot / BS : 0;
  const int off = slot >= 0 ? (int)(slot % BS) : 0;
  // whole-projection norms: one sum of squares over all query entries and
  // one over all key entries
  float inv_q = 1.f, inv_k = 1.f;
  if (ALL && qw != nullptr) {
    float ss = 0.f;
    for (int c = threadIdx.x; c < H * D; c += blockDim.x) {
      const float x = MxElem<T>::ld(q + (size_t)t * ldq + c);
      ss += x * x;
    }
    inv_q = 1.0f / sqrtf(mx_block_sum(ss, red) / (float)(H * D) + eps);
  }
  if (ALL && kw != nullptr) {
    float ss = 0.f;
    for (int c = threadIdx.x; c < G * D; c += blockDim.x) {
      const float x = MxElem<T>::ld(k + (size_t)t * ldk + c);
      ss += x * x;
    }
    inv_k = 1.0f / sqrtf(mx_block_sum(ss, red) / (float)(G * D) + eps);
  }
  for (int hh = wave; hh < H + G; hh += nw) {
    const bool is_q = hh < H;
    const int g = hh - H;
    const T* src = is_q ? q + (size_t)t * ldq + hh * D
                        : k + (size_t)t * ldk + g * D;
    // weight row of this head
    const float* wgt = is_q ? qw : kw;
    if (ALL && wgt != nullptr) wgt += (is_q ? hh : g) * D;
    float inv = is_q ? inv_q : inv_k;
    if (!ALL && wgt != nullptr) {
      float ss = 0.f;
      for (int d = lane; d < D; d += 64) {
        const float x = MxElem<T>::ld(src + d);
        ss += x * x;
      }
      ss = mx_wave_sum(ss);
      inv = 1.0f / sqrtf(ss / (float)D + eps);
    }
    T* dst = nullptr;
    if (is_q) {
      if (wgt != nullptr || csr != nullptr) dst = q + (size_t)t * ldq + hh * D;
    } else if (slot >= 0) {
      dst = kc + ((blk * G + g) * BS + off) * (int64_t)D;
    }
    if (dst == nullptr) continue;
    if (!HALF) {
      for (int d = lane; d < D; d += 64) {
        float x = MxElem<T>::ld(src + d);
        if (wgt != nullptr) x *= inv * wgt[d];
        if (csr != nullptr && d < rot_dims) {
          float y = MxElem<T>::ld(src + (d ^ 1));
          if (wgt != nullptr) y *= inv * wgt[d ^ 1];
          const float* e = csr + (d & ~1);
          x = (d & 1) ? x * e[0] + y * e[1] : x * e[0] - y * e[1];
        }
        MxElem<T>::st(dst + d, x);
      }
    } else {
      const int hd = csr != nullptr ? rot_dims >> 1 : 0;
      for (int i = lane; i < hd; i += 64) {
        float x = MxElem<T>::ld(src + i);
        float y = MxElem<T>::ld(src + i + hd);
        if (wgt != nullptr) {
          x *= inv * wgt[i];
          y *= inv * wgt[i + hd];
        }
        const float c = csr[2 * i], sn = csr[2 * i + 1];
        MxElem<T>::st(dst + i, x * c - y * sn);
        MxElem<T>::st(dst + i + hd, y * c + x * sn);
      }
      for (int d = 2 * hd + lane; d < D; d += 64) {
        float x = MxElem<T>::ld(src + d);
        if (wgt != nullptr) x *= inv * wgt[d];
        MxElem<T>::st(dst + d, x);
      }
    }
  }
  const float lam = vfirst != nullptr ? vmix[0] : 0.f;
  for (int c = threadIdx.x; c < G * DV; c += blockDim.x) {
    float x = MxElem<T>::ld(v + (size_t)t * ldv + c);
    if (vfirst != nullptr) {
      x = (1.0f - lam) * x + lam * MxElem<T>::ld(vfirst + (size_t)t * ldvf + c);
      MxElem<T>::st(v + (size_t)t * ldv + c, x);
    }
    if (slot >= 0) {
      const int g = c / DV, d = c % DV;
      MxElem<T>::st(vc + ((blk * G + g) * BS + off) * (int64_t)DV + d, x);
    }
  }
}

// Pooled keys/values: workgroup (segment, i, column chunk) takes 256
// columns of the i-th block of `pool` positions whose last position this step
// appended (block b covers b*pool .. b*pool + pool - 1) and stores the fp32
// means of its cached keys and values, rounded to the cache type, in the
// pooled caches [NB, G, pr, D|DV]: in the page of the block's first position,
// at row (first position mod BS) div pool. A thread owns one column; its
// loads over the block's positions are independent and run eight at a time.
template <typename T>
__global__ __launch_bounds__(256) void pool_append_kernel(
    const T* __restrict__ kc, const T* __restrict__ vc, T* __restrict__ kp,
    T* __restrict__ vp, const int* __restrict__ block_tables, int max_blocks,
    const int* __restrict__ seq_rows, int G, int D, int DV, int BS, int pool,
    int pr) {
  const int* sr = seq_rows + 4 * blockIdx.x;
  const int n = sr[1], p0 = sr[2];
  const int b = p0 / pool + blockIdx.y;
  if (b >= (p0 + n) / pool) return;
  const int c = blockIdx.z * blockDim.x + threadIdx.x;
  if (c >= G * (D + DV)) return;
  const int* table = block_tables + (size_t)blockIdx.x * max_blocks;
  const int first = b * pool;
  const bool is_k = c < G * D;
  const int cc = is_k ? c : c - G * D;
  const int w = is_k ? D : DV;
  const int g = cc / w, d = cc - g * w;
  const T* cache = (is_k ? kc : vc) + d;
  float acc = 0.f;
  int j = first;
  for (; j + 8 <= first + pool; j += 8) {
    float x[8];
#pragma unroll
    for (int u = 0; u < 8; ++u) {
      const int jj = j + u;
      x[u] = MxElem<T>::ld(
          cache + (((int64_t)table[jj / BS] * G + g) * BS + (jj % BS)) * w);
    }
#pragma unroll
    for (int u = 0; u < 8; ++u) acc += x[u];
  }
  for (; j < first + pool; ++j)
    acc += MxElem<T>::ld(
        cache + (((int64_t)table[j / BS] * G + g) * BS + (j % BS)) * w);
  const int64_t prow =
      ((int64_t)table[first / BS] * G + g) * pr + (first % BS) / pool;
  MxElem<T>::st((is_k ? kp : vp) + prow * w + d, acc / (float)pool);
}

// Queries and keys of attention whose keys are their own values. A group of
// `lanes` lanes (a power of two) takes one head: a query head is divided by
// its root mean square in place, a key head goes to its cache row as it is and
// its 1/rms to kscale [NB, G, BS]. V entries per access; the first one of a
// lane stays in registers between the passes.
template <typename T, int V>
__global__ __launch_bounds__(256) void keyval_prep_kernel(
    T* __restrict__ q, int ldq, const T* __restrict__ k, int ldk, float eps,
    T* __restrict__ cache, float* __restrict__ kscale,
    const int64_t* __restrict__ slots, int H, int G, int D, int BS,
    int lanes) {
  struct __align__(sizeof(T) * V) Vec {
    T e[V];
  };
  const int t = blockIdx.x;
  const int64_t slot = slots[t];
  const int per = blockDim.x / lanes;
  const int gl = threadIdx.x & (lanes - 1), nv = D / V;
  for (int h0 = 0; h0 < H + G; h0 += per) {
    // every lane joins the exchanges below; idle groups repeat the last head
    const int hh = h0 + threadIdx.x / lanes;
    const int hc = min(hh, H + G - 1);
    const bool is_q = hc < H;
    const T* src = is_q ? q + (size_t)t * ldq + (size_t)hc * D
                        : k + (size_t)t * ldk + (size_t)(hc - H) * D;
    float ss = 0.f;
    Vec first;
    for (int c = gl; c < nv; c += lanes) {
      const Vec v = *(const Vec*)(src + c * V);
      if (c == gl) first = v;
#pragma unroll
      for (int i = 0; i < V; ++i) {
        const float x = MxElem<T>::ld(&v.e[i]);
        ss += x * x;
      }
    }
    for (int off = lanes >> 1; off > 0; off >>= 1)
      ss += __shfl_xor(ss, off, 64);
    const float inv = 1.0f / sqrtf(ss / (float)D + eps);
    if (hh >= H + G) continue;
    if (is_q) {
      T* dst = q + (size_t)t * ldq + (size_t)hc * D;
      for (int c = gl; c < nv; c += lanes) {
        Vec v = c == gl ? first : *(const Vec*)(src + c * V);
#pragma unroll
        for (int i = 0; i < V; ++i)
          MxElem<T>::st(&v.e[i], MxElem<T>::ld(&v.e[i]) * inv);
        *(Vec*)(dst + c * V) = v;
      }
    } else if (slot >= 0) {
      const int64_t row = ((slot / BS) * G + (hc - H)) * BS + slot % BS;
      T* dst = cache + row * D;
      for (int c = gl; c < nv; c += lanes)
        *(Vec*)(dst + c * V) = c == gl ? first : *(const Vec*)(src + c * V);
      if (gl == 0) kscale[row] = inv;
    }
  }
}

// Turn the pair (u, w) by the table entry (cos, sin).
PS_DEV void mx_turn(float u, float w, const float* cs, float* ou, float* ow) {
  *ou = u * cs[0] - w * cs[1];
  *ow = w * cs[0] + u * cs[1];
}

// Grid (tokens, 1 + head groups): workgroup y = 0 normalises the latent,
// turns the shared key part and appends the row (nothing to do without dkv:
// the rows are another layer's); workgroup y > 0 assembles the queries of HG
// heads. VEC: latent parts are whole 16-byte vectors. half: the rotary pairs
// are (i, i + rot_dims / 2) instead of neighbours.
#define LP_HG 4

// Entries of pair i of a rotary part of R entries: pairs below rot_dims / 2
// turn; the rest (every pair that lies past rot_dims) passes.
PS_DEV void lp_pair(int i, int rot_dims, int half, int* a, int* b) {
  const int hd = rot_dims >> 1;
  const bool split = half && i < hd;
  *a = split ? i : 2 * i;
  *b = split ? i + hd : 2 * i + 1;
}

template <typename T, bool VEC>
__global__ __launch_bounds__(256) void latent_prep_kernel(
    T* qf, const T* __restrict__ qlat, const T* q, int ldq,
    const T* __restrict__ dkv, int lddkv, const float* __restrict__ normw,
    float eps, const float* __restrict__ cos_sin, int table_rows,
    int rot_dims, const int* __restrict__ positions, T* __restrict__ cache,
    const int64_t* __restrict__ slots, int T_, int H, int D, int R, int L,
    int half) {
  __shared__ float red[17];
  const int t = blockIdx.x;
  const int pos = min(max(positions[t], 0), table_rows - 1);
  const float* cs = cos_sin + (size_t)pos * rot_dims;  // [rot_dims/2][2]
  if (blockIdx.y == 0) {
    if (dkv == nullptr) return;
    const T* row = dkv + (size_t)t * lddkv;
    const int64_t slot = slots[t];
    T* crow = cache + (slot >= 0 ? slot : 0) * (int64_t)(L + R);
    float ss = 0.f;
    for (int c = threadIdx.x; c < L; c += blockDim.x) {
      const float x = MxElem<T>::ld(row + c);
      ss += x * x;
    }
    ss = mx_block_sum(ss, red);
    const float inv = 1.0f / sqrtf(ss / (float)L + eps);
    if (slot < 0) return;
    for (int c = threadIdx.x; c < L; c += blockDim.x)
      MxElem<T>::st(crow + c, MxElem<T>::ld(row + c) * inv * normw[c]);
    // shared key part: pairs below rot_dims turn, the rest passes
    for (int i = threadIdx.x; i < R / 2; i += blockDim.x) {
      int a, b;
      lp_pair(i, rot_dims, half, &a, &b);
      float u = MxElem<T>::ld(row + L + a);
      float w = MxElem<T>::ld(row + L + b);
      if (2 * i < rot_dims) mx_turn(u, w, cs + 2 * i, &u, &w);
      MxElem<T>::st(crow + L + a, u);
      MxElem<T>::st(crow + L + b, w);
    }
    if ((R & 1) && threadIdx.x == 0) crow[L + R - 1] = row[L + R - 1];
    return;
  }
  const int h0 = (blockIdx.y - 1) * LP_HG, hn = min(LP_HG, H - h0);
  if (qlat == nullptr) {
    // queries stay as they are, their rotary parts turn in place (qf is q);
    // a thread owns both entries of a pair
    for (int c = threadIdx.x; c < hn * (rot_dims / 2); c += blockDim.x) {
      const int h = c / (rot_dims / 2), i = c - h * (rot_dims / 2);
      T* p = qf + (size_t)t * ldq + (h0 + h) * (D + R) + D;
      int a, b;
      lp_pair(i, rot_dims, half, &a, &b);
      float u, w;
      mx_turn(MxElem<T>::ld(p + a), MxElem<T>::ld(p + b), cs + 2 * i, &u, &w);
      MxElem<T>::st(p + a, u);
      MxElem<T>::st(p + b, w);
    }
    return;
  }
  // queries: per head [latent-space part | turned rotary part]
  const int QW = L + R;
  T* qrow = qf + (size_t)t * H * QW + (size_t)h0 * QW;
  if (VEC) {
    constexpr int V = 16 / sizeof(T);
    const int n = L / V;
    for (int c = threadIdx.x; c < hn * n; c += blockDim.x) {
      const int h = c / n, l = (c - h * n) * V;
      *(uint4*)(qrow + h * QW + l) =
          *(const uint4*)(qlat + ((size_t)(h0 + h) * T_ + t) * L + l);
    }
  } else {
    for (int c = threadIdx.x; c < hn * L; c += blockDim.x) {
      const int h = c / L, l = c - h * L;
      qrow[h * QW + l] = qlat[((size_t)(h0 + h) * T_ + t) * L + l];
    }
  }
  for (int c = threadIdx.x; c < hn * (R / 2); c += blockDim.x) {
    const int h = c / (R / 2), i = c - h * (R / 2);
    const T* src = q + (size_t)t * ldq + (h0 + h) * (D + R) + D;
    int a, b;
    lp_pair(i, rot_dims, half, &a, &b);
    float u = MxElem<T>::ld(src + a);
    float w = MxElem<T>::ld(src + b);
    if (2 * i < rot_dims) mx_turn(u, w, cs + 2 * i, &u, &w);
    T* dst = qrow + h * QW + L;
    MxElem<T>::st(dst + a, u);
    MxElem<T>::st(dst + b, w);
  }
  if (R & 1)
    for (int h = threadIdx.x; h < hn; h += blockDim.x)
      qrow[h * QW + QW - 1] =
          q[(size_t)t * ldq + (h0 + h) * (D + R) + D + R - 1];
}

// y[t] = x[t] / sqrt(mean(x[t]^2) + eps) * w. One workgroup per row.
template <typename T>
__global__ __launch_bounds__(256) void rms_norm_rows_kernel(
    T* __restrict__ y, const T* __restrict__ x, int ldx,
    const float* __restrict__ w, float eps, int C) {
  __shared__ float red[17];
  const T* xr = x + (size_t)blockIdx.x * ldx;
  T* yr = y + (size_t)blockIdx.x * C;
  float ss = 0.f;
  for (int c = threadIdx.x; c < C; c += blockDim.x) {
    const float v = MxElem<T>::ld(xr + c);
    ss += v * v;
  }
  const float inv = 1.0f / sqrtf(mx_block_sum(ss, red) / (float)C + eps);
  for (int c = threadIdx.x; c < C; c += blockDim.x)
    MxElem<T>::st(yr + c, MxElem<T>::ld(xr + c) * inv * w[c]);
}

// out[t, h*DV + d] = o[h*hs + t*rs + d] * sigmoid(gate[t, h]) (gate nullptr:
// the plain copy). out may be o itself where both lie the same way. Grid (column chunks, tokens); a thread takes V consecutive
// entries of one head (V divides DV).
template <typename T, int V>
__global__ __launch_bounds__(256) void merge_heads_kernel(
    T* out, int ldo, const T* o, int64_t hs, int64_t rs,
    const T* __restrict__ gate, int ldg, int H, int DV) {
  const int t = blockIdx.y;
  const int c = (blockIdx.x * blockDim.x + threadIdx.x) * V;
  if (c >= H * DV) return;
  const int h = c / DV, d = c - h * DV;
  const T* src = o + h * hs + t * rs + d;
  T* dst = out + (size_t)t * ldo + c;
  const float g = gate != nullptr
                      ? mx_sigmoid(MxElem<T>::ld(gate + (size_t)t * ldg + h))
                      : 1.f;
  struct __align__(sizeof(T) * V) Vec {
    T e[V];
  };
  const Vec v = *(const Vec*)src;
  Vec r;
#pragma unroll
  for (int i = 0; i < V; ++i) MxElem<T>::st(&r.e[i], MxElem<T>::ld(&v.e[i]) * g);
  *(Vec*)dst = r;
}

// One wave per row: segment blockIdx.y's row r comes from position p0 + r of
// its sequence; the rows up to the next multiple of `pad` are zero-filled.
// U: copy unit.
template <typename U>
__global__ __launch_bounds__(256) void latent_gather_kernel(
    U* __restrict__ out, const U* __restrict__ cache,
    const int* __restrict__ block_tables, int max_blocks,
    const int* __restrict__ segments, int BS, int units, int pad) {
  const int* sg = segments + 3 * blockIdx.y;
  const int r = blockIdx.x * 4 + (threadIdx.x >> 6);
  if (r >= sg[1]) {
    if (r < (sg[1] + pad - 1) / pad * pad) {
      U* dst = out + ((int64_t)sg[0] + r) * units;
      for (int c = threadIdx.x & 63; c < units; c += 64) dst[c] = U();
    }
    return;
  }
  const int p = sg[2] + r;
  const int blk = block_tables[(size_t)blockIdx.y * max_blocks + p / BS];
  const U* src = cache + ((int64_t)blk * BS + p % BS) * units;
  U* dst = out + ((int64_t)sg[0] + r) * units;
  for (int c = threadIdx.x & 63; c < units; c += 64) dst[c] = src[c];
}

// Thread = channel, workgroup = (channel tile, segment, chunk of CONV_CH
// tokens). A thread keeps the K-1 inputs before its current token in
// registers. Only chunk 0 of a segment reads the sequence's state, and it
// writes the new state (the segment's last K-1 inputs) afterwards, so no
// other workgroup races with it.
#define CONV_CH 64

template <typename T, int K>
__global__ __launch_bounds__(256) void short_conv_silu_kernel(
    T* __restrict__ y, int ldy, const T* __restrict__ x, int ldx,
    const float* __restrict__ w, const float* __restrict__ bias,
    T* __restrict__ state, const int* __restrict__ seq_rows, int C) {
  const int c = blockIdx.x * blockDim.x + threadIdx.x;
  const int* sr = seq_rows + 4 * blockIdx.y;
  const int t0 = sr[0], n = sr[1], p0 = sr[2], slot = sr[3];
  const int a = blockIdx.z * CONV_CH;
  if (c >= C || a >= n) return;
  const int b = min(n, a + CONV_CH);
  constexpr int P = K > 1 ? K - 1 : 1;
  float wk[K], win[P], old[P];
#pragma unroll
  for (int j = 0; j < K; ++j) wk[j] = w[(size_t)c * K + j];
  const float b0 = bias != nullptr ? bias[c] : 0.f;
  T* st = state + (size_t)slot * (K - 1) * C;
#pragma unroll
  for (int j = 0; j < K - 1; ++j) {
    const int r = a - (K - 1) + j;  // row of the segment, < 0: before it
    if (r >= 0)
      win[j] = MxElem<T>::ld(x + (size_t)(t0 + r) * ldx + c);
    else
      win[j] = p0 > 0 ? MxElem<T>::ld(st + (size_t)(K - 1 + r) * C + c) : 0.f;
    old[j] = win[j];
  }
  for (int t = a; t < b; ++t) {
    const float cur = MxElem<T>::ld(x + (size_t)(t0 + t) * ldx + c);
    float acc = b0 + wk[K - 1] * cur;
#pragma unroll
    for (int j = 0; j < K - 1; ++j) acc += wk[j] * win[j];
#pragma unroll
    for (int j = 0; j + 1 < K - 1; ++j) win[j] = win[j + 1];
    if (K > 1) win[K - 2] = cur;
    MxElem<T>::st(y + (size_t)(t0 + t) * ldy + c, acc * mx_sigmoid(acc));
  }
  if (a == 0) {
    // old[] holds the previous state (a == 0: rows -(K-1) .. -1)
#pragma unroll
    for (int j = 0; j < K - 1; ++j) {
      const int r = n - (K - 1) + j;
      float val;
      if (r >= 0) {
        val = MxElem<T>::ld(x + (size_t)(t0 + r) * ldx + c);
      } else {
        val = 0.f;
#pragma unroll
        for (int e = 0; e < K - 1; ++e)
          if (e == K - 1 + r) val = old[e];
      }
      MxElem<T>::st(st + (size_t)j * C + c, val);
    }
  }
}

extern "C" {

void mx_attn_prep(void* q, int ldq, const void* k, int ldk, void* v, int ldv,
                  const void* qw, const void* kw, float eps, const void* vmix,
                  const void* vfirst, int ldvf, void* kc, void* vc,
                  const void* slots, int T_, int H, int G, int D, int DV,
                  int BS, const void* cos_sin, int table_rows, int rot_dims,
                  const void* positions, int norm_all, int half, int dtype,
                  void* stream) {
  if (T_ <= 0) return;
#define AP_GO(HALF_, ALL_)                                                  \
  hipLaunchKernelGGL((attn_prep_kernel<T, HALF_, ALL_>), dim3(T_), dim3(256), \
                     0, (hipStream_t)stream, (T*)q, ldq, (const T*)k, ldk,   \
                     (T*)v, ldv, (const float*)qw, (const float*)kw, eps,    \
                     (const float*)vmix, (const T*)vfirst, ldvf, (T*)kc,     \
                     (T*)vc, (const int64_t*)slots, H, G, D, DV, BS,         \
                     (const float*)cos_sin, table_rows, rot_dims,            \
                     (const int*)positions)
  MX_DISPATCH_DTYPE(dtype, {
    if (half && norm_all) AP_GO(true, true);
    else if (half) AP_GO(true, false);
    else if (norm_all) AP_GO(false, true);
    else AP_GO(false, false);
  })
#undef AP_GO
}

void mx_keyval_prep(void* q, int ldq, const void* k, int ldk, float eps,
                    void* cache, void* kscale, const void* slots, int T_,
                    int H, int G, int D, int BS, int dtype, void* stream) {
  if (T_ <= 0 || H <= 0 || G <= 0 || D <= 0) return;
  const bool aligned = (((size_t)q | (size_t)k | (size_t)cache) & 15) == 0;
#define KP_GO(V)                                                             \
  {                                                                          \
    int lanes = 1;                                                           \
    while (lanes < 64 && lanes * (V) < D) lanes <<= 1;                       \
    hipLaunchKernelGGL((keyval_prep_kernel<T, V>), dim3(T_), dim3(256), 0,   \
                       (hipStream_t)stream, (T*)q, ldq, (const T*)k, ldk,    \
                       eps, (T*)cache, (float*)kscale,                       \
                       (const int64_t*)slots, H, G, D, BS, lanes);           \
  }
  MX_DISPATCH_DTYPE(dtype, {
    constexpr int VN = 16 / sizeof(T);
    if (aligned && D % VN == 0 && ldq % VN == 0 && ldk % VN == 0)
      KP_GO(VN)
    else
      KP_GO(1)
  })
#undef KP_GO
}

void mx_pool_append(const void* kc, const void* vc, void* kp, void* vp,
                    const void* block_tables, int max_blocks,
                    const void* seq_rows, int S_, int blocks_per_seg, int G,
                    int D, int DV, int BS, int pool, int dtype,
                    void* stream) {
  if (S_ <= 0 || blocks_per_seg <= 0 || pool < 1) return;
  const int pr = (BS + pool - 1) / pool;
  MX_DISPATCH_DTYPE(dtype, {
    hipLaunchKernelGGL((pool_append_kernel<T>),
                       dim3(S_, blocks_per_seg, (G * (D + DV) + 255) / 256),
                       dim3(256), 0, (hipStream_t)stream, (const T*)kc,
                       (const T*)vc, (T*)kp, (T*)vp,
                       (const int*)block_tables, max_blocks,
                       (const int*)seq_rows, G, D, DV, BS, pool, pr);
  })
}

void mx_latent_prep(void* qf, const void* qlat, const void* q, int ldq,
                    const void* dkv, int lddkv, const void* normw, float eps,
                    const void* cos_sin, int table_rows, int rot_dims,
                    const void* positions, void* cache, const void* slots,
                    int T_, int H, int D, int R, int L, int BS, int half,
                    int dtype, void* stream) {
  if (T_ <= 0) return;
  (void)BS;
  dim3 grid(T_, 1 + (H + LP_HG - 1) / LP_HG);
#define LP_GO(VEC)                                                           \
  hipLaunchKernelGGL((latent_prep_kernel<T, VEC>), grid, dim3(256), 0,       \
                     (hipStream_t)stream, (T*)qf, (const T*)qlat,            \
                     (const T*)q, ldq, (const T*)dkv, lddkv,                 \
                     (const float*)normw, eps, (const float*)cos_sin,        \
                     table_rows, rot_dims, (const int*)positions, (T*)cache, \
                     (const int64_t*)slots, T_, H, D, R, L, half)
  MX_DISPATCH_DTYPE(dtype, {
    constexpr int V = 16 / sizeof(T);
    const bool vec = L % V == 0 && (L + R) % V == 0 &&
                     (((size_t)qf | (size_t)qlat) & 15) == 0;
    if (vec)
      LP_GO(true);
    else
      LP_GO(false);
  })
#undef LP_GO
}

void mx_rms_norm_rows(void* y, const void* x, int ldx, const void* w,
                      float eps, int T_, int C, int dtype, void* stream) {
  if (T_ <= 0 || C <= 0) return;
  MX_DISPATCH_DTYPE(dtype, {
    hipLaunchKernelGGL((rms_norm_rows_kernel<T>), dim3(T_), dim3(256), 0,
                       (hipStream_t)stream, (T*)y, (const T*)x, ldx,
                       (const float*)w, eps, C);
  })
}

void mx_merge_heads(void* out, int ldo, const void* o, int hs, int rs,
                    const void* gate, int ldg, int T_, int H, int DV,
                    int dtype, void* stream) {
  if (T_ <= 0 || H * DV <= 0) return;
  const bool aligned = (((size_t)out | (size_t)o) & 15) == 0;
  MX_DISPATCH_DTYPE(dtype, {
    constexpr int V = 16 / sizeof(T);
    if (aligned && DV % V == 0 && ldo % V == 0 && hs % V == 0 &&
        rs % V == 0) {
      hipLaunchKernelGGL((merge_heads_kernel<T, V>),
                         dim3((H * DV / V + 255) / 256, T_), dim3(256), 0,
                         (hipStream_t)stream, (T*)out, ldo, (const T*)o,
                         (int64_t)hs, (int64_t)rs, (const T*)gate, ldg, H,
                         DV);
    } else {
      hipLaunchKernelGGL((merge_heads_kernel<T, 1>),
                         dim3((H * DV + 255) / 256, T_), dim3(256), 0,
                         (hipStream_t)stream, (T*)out, ldo, (const T*)o,
                         (int64_t)hs, (int64_t)rs, (const T*)gate, ldg, H,
                         DV);
    }
  })
}

void mx_latent_gather(void* out, const void* cache, const void* block_tables,
                      int max_blocks, const void* segments, int S_,
                      int longest, int BS, int D, int pad, int dtype,
                      void* stream) {
  if (S_ <= 0 || longest <= 0 || pad < 1) return;
  const int bytes = D * (dtype == MX_BF16 ? 2 : 4);
  dim3 grid(((longest + pad - 1) / pad * pad + 3) / 4, S_);
#define LG_GO(U)                                                            \
  hipLaunchKernelGGL((latent_gather_kernel<U>), grid, dim3(256), 0,         \
                     (hipStream_t)stream, (U*)out, (const U*)cache,         \
                     (const int*)block_tables, max_blocks,                  \
                     (const int*)segments, BS, bytes / (int)sizeof(U), pad)
  if (bytes % 16 == 0 && (((size_t)out | (size_t)cache) & 15) == 0)
    LG_GO(uint4);
  else
    LG_GO(unsigned short);
#undef LG_GO
}

#define CONV_CASE(KK)                                                        \
  case KK:                                                                   \
    hipLaunchKernelGGL((short_conv_silu_kernel<T, KK>), grid, dim3(256), 0,  \
                       (hipStream_t)stream, (T*)y, ldy, (const T*)x, ldx,    \
                       (const float*)w, (const float*)bias, (T*)state,       \
                       (const int*)seq_rows, C);                             \
    break;

int mx_short_conv_silu(void* y, int ldy, const void* x, int ldx,
                       const void* w, const void* bias, void* state,
                       const void* seq_rows,
                       int S_, int C, int K, int T_, int dtype,
                       void* stream) {
  if (S_ <= 0 || T_ <= 0) return 0;
  if (K < 1 || K > 8) return 1;
  // a segment has at most T_ - (S_ - 1) rows
  const int longest = T_ - (S_ - 1);
  dim3 grid((C + 255) / 256, S_, (longest + CONV_CH - 1) / CONV_CH);
  MX_DISPATCH_DTYPE(dtype, {
    switch (K) {
      CONV_CASE(1)
      CONV_CASE(2)
      CONV_CASE(3)
      CONV_CASE(4)
      CONV_CASE(5)
      CONV_CASE(6)
      CONV_CASE(7)
      CONV_CASE(8)
    }
  })
  return 0;
}

}  // extern "C"
