// Linear attention with one fixed decay per head (gfx950):
//
//   S_t = a_h S_{t-1} + k_t v_t^T,   o_t = S_t^T q_t        S [N, P] fp32
//
// q, k and v arrive as projected and pass silu here (SILU).  Two kernels:
//
//   step    any type and sizes, any number of rows: a workgroup keeps 64
//           columns of S in registers (16 threads x 4 columns, 16 groups of
//           key entries), so one decoded row is one load, one update and
//           one store of the state with every access 16 bytes wide and all
//           of them in flight together.
//   chunks  bf16, N <= 128, MFMA: rows in chunks of C = 64.  With L rows
//           in the chunk and S the memory before it,
//             O[i] = a^{i+1} q_i S + sum_{j <= i} a^{i-j} (q_i.k_j) v_j
//             S   <- a^L S + sum_j k_j (a^{L-1-j} v_j)^T
//           A wave owns 16 value columns and keeps S for them as MFMA
//           accumulators (fp32, in registers) across all chunks; S^T as the
//           next product's operand, the weighted scores a^{i-j} (q.k) and
//           the decayed values enter the matrix cores as a bf16 pair (high
//           part + remainder), 16 mantissa bits, so recurrent state and
//           attention weights are not rounded to bf16.
//
// The order of a contraction index is free as long as both operands agree
// on it: accumulator tiles (lane = column, 4 consecutive rows) of two
// neighbouring tiles are used directly as an operand of 32 contraction
// entries, with lane group g holding entries {4g..4g+3, 16+4g..16+4g+3};
// the other operand is fetched from LDS in that order (two 8-byte reads).
//
// Long prompts of few sequences are cut into segments: a first launch
// leaves every segment's own contribution k (a^.. v)^T, a second one turns
// these into the memory at each segment's start (and the sequence's final
// state), and the main launch then runs all segments side by side.
#include "../csrc_hybrid/act_types.h"

namespace igw {

typedef __attribute__((ext_vector_type(8))) short fd_short8;
typedef __attribute__((ext_vector_type(4))) short fd_short4;
typedef __attribute__((ext_vector_type(4))) float fd_float4;

// round to nearest even by the conversion instruction
DEVINLINE uint16_t cvt_bf16(float x) {
  return __builtin_bit_cast(uint16_t, (__bf16)x);
}

// two at a time: one instruction
typedef __attribute__((ext_vector_type(2))) float fd_float2;
typedef __attribute__((ext_vector_type(2))) __bf16 fd_bf2;
typedef __attribute__((ext_vector_type(2))) unsigned short fd_ushort2;
DEVINLINE fd_ushort2 cvt_bf16x2(float a, float b) {
  return __builtin_bit_cast(
      fd_ushort2, __builtin_convertvector(fd_float2{a, b}, fd_bf2));
}

// silu as the activation type holds it: both kernels see the same values
template <typename T>
DEVINLINE float silu_act(float z);
template <>
DEVINLINE float silu_act<float>(float z) {
  return z * sigmoid_f32(z);
}
DEVINLINE float silu_fast(float z) {
  return z * __builtin_amdgcn_rcpf(1.0f + __expf(-z));
}
template <>
DEVINLINE float silu_act<uint16_t>(float z) {
  return bf16_to_f32(cvt_bf16(silu_fast(z)));
}

// ---------------------------------------------------------------------------
// step kernel
// ---------------------------------------------------------------------------
constexpr int FD_ROWS = 16;   // rows of q, k, v staged at a time
constexpr int FD_PT = 64;     // value columns per workgroup

template <typename T, int NPER, bool V4>
__global__ __launch_bounds__(256) void fixed_decay_step_kernel(
    float* __restrict__ out, const T* __restrict__ q, int64_t q_s0,
    int64_t q_s1, const T* __restrict__ k, int64_t k_s0, int64_t k_s1,
    const T* __restrict__ v, int64_t v_s0, int64_t v_s1,
    const float* __restrict__ decay, float* __restrict__ state,
    const int32_t* __restrict__ seqs, const int32_t* __restrict__ seq_cu,
    const int32_t* __restrict__ seq_start,
    const int32_t* __restrict__ seq_slots, int H, int G, int N, int P,
    int silu) {
  // q rows | k rows | v rows (FD_PT columns) | partial read-outs
  extern __shared__ __attribute__((aligned(16))) float lds[];
  float* lq = lds;
  float* lk = lq + FD_ROWS * N;
  float* lv = lk + FD_ROWS * N;
  float* red = lv + FD_ROWS * FD_PT;      // [2][4 waves][FD_PT]
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  const int h = blockIdx.y, s = seqs[blockIdx.z];
  const int g = h / (H / G);
  const int r0 = seq_cu[s], r1 = seq_cu[s + 1];
  if (r1 == r0) return;
  const int c4 = (tid & 15) * 4, ng = tid >> 4;
  const int p0 = blockIdx.x * FD_PT, p = p0 + c4;
  const float a = decay[h];
  const bool fresh = seq_start[s] == 0;
  float* st = state + ((int64_t)seq_slots[s] * H + h) * N * P;

  float S[NPER][4];
#pragma unroll
  for (int i = 0; i < NPER; ++i) {
    const int n = i * 16 + ng;
#pragma unroll
    for (int e = 0; e < 4; ++e) S[i][e] = 0.0f;
    if (fresh || n >= N) continue;
    if (V4) {
      if (p < P) {
        const float4 x = *(const float4*)(st + (int64_t)n * P + p);
        S[i][0] = x.x;
        S[i][1] = x.y;
        S[i][2] = x.z;
        S[i][3] = x.w;
      }
    } else {
#pragma unroll
      for (int e = 0; e < 4; ++e)
        if (p + e < P) S[i][e] = st[(int64_t)n * P + p + e];
    }
  }
  int par = 0;
  for (int c0 = r0; c0 < r1; c0 += FD_ROWS) {
    const int tc = min(FD_ROWS, r1 - c0);
    if (c0 != r0) __syncthreads();    // everybody is done with the last rows
    for (int i = tid; i < tc * N; i += 256) {
      const int t = i / N, n = i - t * N;
      const float x = Act<T>::ld(q + (c0 + t) * q_s0 + g * q_s1 + n);
      const float y = Act<T>::ld(k + (c0 + t) * k_s0 + g * k_s1 + n);
      lq[i] = silu ? silu_act<T>(x) : x;
      lk[i] = silu ? silu_act<T>(y) : y;
    }
    for (int i = tid; i < tc * FD_PT; i += 256) {
      const int t = i / FD_PT, c = i - t * FD_PT;
      float x = 0.0f;
      if (p0 + c < P) {
        x = Act<T>::ld(v + (c0 + t) * v_s0 + h * v_s1 + p0 + c);
        if (silu) x = silu_act<T>(x);
      }
      lv[i] = x;
    }
    __syncthreads();
    for (int t = 0; t < tc; ++t) {
      const float4 vv = *(const float4*)(lv + t * FD_PT + c4);
      float o[4] = {0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
      for (int i = 0; i < NPER; ++i) {
        const int n = i * 16 + ng;
        if (n >= N) continue;
        const float kn = lk[t * N + n], qn = lq[t * N + n];
        S[i][0] = a * S[i][0] + kn * vv.x;
        S[i][1] = a * S[i][1] + kn * vv.y;
        S[i][2] = a * S[i][2] + kn * vv.z;
        S[i][3] = a * S[i][3] + kn * vv.w;
#pragma unroll
        for (int e = 0; e < 4; ++e) o[e] += qn * S[i][e];
      }
      // sum over the four groups of a wave, then over the waves.  Two
      // buffers in turn: a buffer is written again only after the next
      // row's barrier, which its readers reach when they have read it
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        o[e] += __shfl_xor(o[e], 16, 64);
        o[e] += __shfl_xor(o[e], 32, 64);
      }
      float* rb = red + par * 4 * FD_PT;
      if (lane < 16)
        *(float4*)(rb + wave * FD_PT + c4) =
            make_float4(o[0], o[1], o[2], o[3]);
      __syncthreads();
      if (tid < FD_PT && p0 + tid < P)
        out[((int64_t)(c0 + t) * H + h) * P + p0 + tid] =
            rb[tid] + rb[FD_PT + tid] + rb[2 * FD_PT + tid] +
            rb[3 * FD_PT + tid];
      par ^= 1;
    }
  }
#pragma unroll
  for (int i = 0; i < NPER; ++i) {
    const int n = i * 16 + ng;
    if (n >= N) continue;
    if (V4) {
      if (p < P)
        *(float4*)(st + (int64_t)n * P + p) =
            make_float4(S[i][0], S[i][1], S[i][2], S[i][3]);
    } else {
#pragma unroll
      for (int e = 0; e < 4; ++e)
        if (p + e < P) st[(int64_t)n * P + p + e] = S[i][e];
    }
  }
}

// ---------------------------------------------------------------------------
// chunk kernel
// ---------------------------------------------------------------------------
constexpr int FD_C = 64;      // rows per chunk

// 8 floats -> bf16 high parts and bf16 remainders
DEVINLINE void split_pair(const float* x, fd_short8& hi, fd_short8& lo) {
#pragma unroll
  for (int e = 0; e < 8; e += 2) {
    const fd_ushort2 b = cvt_bf16x2(x[e], x[e + 1]);
    const fd_ushort2 r = cvt_bf16x2(x[e] - bf16_to_f32(b[0]),
                                    x[e + 1] - bf16_to_f32(b[1]));
    hi[e] = (short)b[0];
    hi[e + 1] = (short)b[1];
    lo[e] = (short)r[0];
    lo[e + 1] = (short)r[1];
  }
}

DEVINLINE fd_float4 mfma_bf16(fd_short8 a, fd_short8 b, fd_float4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0);
}

// The transposed tiles hold FD_C rows of the chunk per key entry or value
// column: 128 bytes, eight 16-byte pieces, piece c of row n stored at c ^
// (n & 7) ^ (n >> 3 & 7).  Staging lanes write rows that are 8 apart,
// operand reads touch 16 neighbouring rows: either way the lanes spread
// over all banks.
// Row n = 16 t + m (m < 16): t enters the piece by itself, so a lane's
// address is one exclusive-or away from that of t = 0.
DEVINLINE int fd_swz(int t, int m, int j) {
  return t * 16 * FD_C + m * FD_C +
         ((((j >> 3) ^ m ^ (m >> 3) ^ (2 * t)) & 7) << 3) + (j & 7);
}

// Rows of q and k (NP entries): piece c at c ^ a row number that changes
// every 256 bytes, for operand reads of 16 neighbouring rows.
// Row j = 16 t + m: the piece depends on m alone.
template <int NP>
DEVINLINE int fd_row(int t, int m, int n) {
  return t * 16 * NP + m * NP +
         ((((n >> 3) ^ (m / (128 / NP))) & (NP / 8 - 1)) << 3) + (n & 7);
}

// entries {j0 + 4g ..} and {j0 + 16 + 4g ..} of four each
DEVINLINE fd_short8 fd_join(fd_short4 a, fd_short4 b) {
  return fd_short8{a[0], a[1], a[2], a[3], b[0], b[1], b[2], b[3]};
}

// segment table, int32 [5][nseg]: first row, end row, sequence, first
// segment of its sequence (0/1), last segment of its sequence (0/1)
template <int NP, int NW, bool VEC, bool STATE_ONLY>
__global__ __launch_bounds__(NW * 64, NW / 2) void fixed_decay_chunk_kernel(
    float* __restrict__ out, const uint16_t* __restrict__ q, int64_t q_s0,
    int64_t q_s1, const uint16_t* __restrict__ k, int64_t k_s0, int64_t k_s1,
    const uint16_t* __restrict__ v, int64_t v_s0, int64_t v_s1,
    const float* __restrict__ decay, float* __restrict__ state,
    float* __restrict__ work, const int32_t* __restrict__ segs, int nseg,
    const int32_t* __restrict__ seq_start,
    const int32_t* __restrict__ seq_slots, int H, int G, int N, int P,
    int silu) {
  constexpr int NTILE = NP / 16;
  constexpr int PT = NW * 16;
  constexpr int NQ = NP / 8 / NW > 0 ? NP / 8 / NW : 1;   // pieces per thread
  constexpr int PG = NP / 8 < 8 ? NP / 8 : 8;   // neighbouring lanes' pieces
  __shared__ __attribute__((aligned(16))) uint16_t qs[STATE_ONLY ? 8
                                                                 : FD_C * NP];
  __shared__ __attribute__((aligned(16))) uint16_t ks[STATE_ONLY ? 8
                                                                 : FD_C * NP];
  __shared__ __attribute__((aligned(16))) uint16_t kt[NP * FD_C];
  __shared__ __attribute__((aligned(16))) uint16_t vt[PT * FD_C];
  // weighted scores as operand fragments [hi|lo][lane]: row tiles 0-3
  // against rows 0-31, then row tiles 2-3 against rows 32-63
  __shared__ __attribute__((aligned(16)))
  uint16_t af[STATE_ONLY ? 8 : 6 * 2 * 64 * 8];
  // powers of the decay behind as many zeros: pw[negative] = 0
  __shared__ float pw_lds[2 * FD_C + 1];
  float* pw = pw_lds + FD_C;
  int tid = threadIdx.x;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int lane = tid & 63;
  int l16 = lane & 15, g4 = lane >> 4;
  const int sg = blockIdx.z, h = blockIdx.y;
  const int row0 = segs[sg], row1 = segs[nseg + sg];
  const int seq = segs[2 * nseg + sg];
  const bool first = segs[3 * nseg + sg] != 0;
  const bool last = segs[4 * nseg + sg] != 0;
  const int kh = h / (H / G);
  const float a = decay[h];
  for (int i = tid; i <= 2 * FD_C; i += NW * 64) {
    const int e = i - FD_C;
    pw_lds[i] = e < 0 ? 0.0f : e == 0 ? 1.0f : powf(a, (float)e);
  }
  const int p0 = blockIdx.x * PT;
  const int pc = p0 + wave * 16 + l16;     // this lane's value column
  float* st = state + ((int64_t)seq_slots[seq] * H + h) * N * P;
  float* wk = work == nullptr
                  ? nullptr
                  : work + ((int64_t)sg * H + h) * N * P;

  // S tiles: column pc, rows 16 nt + 4 g4 + r
  fd_float4 S[NTILE];
  {
    const float* src = nullptr;
    if (!STATE_ONLY) {
      if (wk != nullptr) src = wk;                 // memory at its start
      else if (!(first && seq_start[seq] == 0)) src = st;
    }
#pragma unroll
    for (int nt = 0; nt < NTILE; ++nt)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int n = nt * 16 + g4 * 4 + r;
        S[nt][r] = (src != nullptr && n < N && pc < P)
                       ? src[(int64_t)n * P + pc]
                       : 0.0f;
      }
  }

  // staging: PG (values: 8) neighbouring lanes take neighbouring pieces of
  // 8 entries of one row, so a row's 128 bytes arrive in one request
  ushort8 qr[NQ], kr[NQ], vr[2];
  auto piece = [&](const uint16_t* base, int width, int c8, bool ok) {
    ushort8 x;
#pragma unroll
    for (int e = 0; e < 8; ++e) x.v[e] = 0;
    if (!ok) return x;
    if (VEC) {
      if (c8 < width) x = *(const ushort8*)(base + c8);
    } else {
#pragma unroll
      for (int e = 0; e < 8; ++e)
        if (c8 + e < width) x.v[e] = base[c8 + e];
    }
    return x;
  };
  auto k_place = [&](int i, int& j, int& c8) {
    const int idx = tid + i * NW * 64;
    j = (idx / PG) & (FD_C - 1);
    c8 = (idx / (PG * FD_C) * PG + (idx & (PG - 1))) * 8;
  };
  auto v_place = [&](int i, int& j, int& c8) {
    const int idx = tid + i * NW * 64;
    j = (idx >> 3) & (FD_C - 1);
    c8 = ((idx >> 9) * 8 + (idx & 7)) * 8;
  };
  // one base per chunk for the whole workgroup, 32-bit offsets per lane
  const int ks0 = (int)k_s0, qs0 = (int)q_s0, vs0 = (int)v_s0;
  auto fetch = [&](int c0) {
    const uint16_t* kb = k + (int64_t)c0 * k_s0 + kh * k_s1;
    const uint16_t* qb = q + (int64_t)c0 * q_s0 + kh * q_s1;
    const uint16_t* vb = v + (int64_t)c0 * v_s0 + h * v_s1 + p0;
    const int left = row1 - c0;
    int j, c8;
#pragma unroll
    for (int i = 0; i < NQ; ++i) {
      k_place(i, j, c8);
      const bool in = j < left && c8 < NP;
      kr[i] = piece(kb + j * ks0, N, c8, in);
      if (!STATE_ONLY) qr[i] = piece(qb + j * qs0, N, c8, in);
    }
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      v_place(i, j, c8);
      vr[i] = piece(vb + j * vs0, P - p0, c8, j < left);
    }
  };
  // eight entries of row j, transposed, from column c8 on (a multiple of 8)
  auto put8 = [&](uint16_t* tile, int c8, int j, ushort8 x) {
    const int at = c8 * FD_C + ((((j >> 3) ^ (c8 >> 3)) & 7) << 3) + (j & 7);
#pragma unroll
    for (int e = 0; e < 8; ++e) tile[(at ^ (e << 3)) + e * FD_C] = x.v[e];
  };
  auto act8 = [&](ushort8 x) {
    if (silu) {
#pragma unroll
      for (int e = 0; e < 8; e += 2) {
        const fd_ushort2 y = cvt_bf16x2(silu_fast(bf16_to_f32(x.v[e])),
                                        silu_fast(bf16_to_f32(x.v[e + 1])));
        x.v[e] = y[0];
        x.v[e + 1] = y[1];
      }
    }
    return x;      // silu(0) = 0: padding stays zero
  };

  fetch(row0);
  for (int c0 = row0; c0 < row1; c0 += FD_C) {
    const int L = min(FD_C, row1 - c0);
    // LDS addresses are recomputed per chunk: kept across chunks they would
    // cost half of the registers
    if (NW == 8) asm volatile("" : "+v"(tid), "+v"(l16), "+v"(g4));
    int j, c8;
#pragma unroll
    for (int i = 0; i < NQ; ++i) {
      k_place(i, j, c8);
      if (c8 < NP) {
        const ushort8 kk = act8(kr[i]);
        put8(kt, c8, j, kk);
        if (!STATE_ONLY) {
          const int at = fd_row<NP>(j >> 4, j & 15, c8);
          *(ushort8*)(ks + at) = kk;
          *(ushort8*)(qs + at) = act8(qr[i]);
        }
      }
    }
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      v_place(i, j, c8);
      put8(vt, c8, j, act8(vr[i]));
    }
    __syncthreads();
    if (NW == 4 && c0 + FD_C < row1) fetch(c0 + FD_C);

    if (!STATE_ONLY) {
      // weighted scores of (16 rows i) x (32 rows j), transposed product
      // K Q^T: lane column = i, accumulator rows = j
      for (int un = wave; un < 8; un += NW) {
        const int it = un & 3, kst = un >> 2;
        if (kst * 32 > it * 16 + 15) continue;     // all j > i
        fd_float4 c[2];
#pragma unroll
        for (int x = 0; x < 2; ++x) c[x] = fd_float4{0, 0, 0, 0};
#pragma unroll
        for (int ns = 0; ns < NP / 32; ++ns) {
          const fd_short8 b = *(const fd_short8*)(
              qs + fd_row<NP>(it, l16, ns * 32 + g4 * 8));
#pragma unroll
          for (int x = 0; x < 2; ++x) {
            const fd_short8 aa = *(const fd_short8*)(
                ks + fd_row<NP>(kst * 2 + x, l16, ns * 32 + g4 * 8));
            c[x] = mfma_bf16(aa, b, c[x]);
          }
        }
        // a^{i-j}, zero for j > i
        float w[8];
        const float* pij = pw + it * 16 + l16 - kst * 32 - g4 * 4;
#pragma unroll
        for (int x = 0; x < 2; ++x)
#pragma unroll
          for (int r = 0; r < 4; ++r)
            w[x * 4 + r] = pij[-(x * 16 + r)] * c[x][r];
        fd_short8 hi, lo;
        split_pair(w, hi, lo);
        uint16_t* f = af + ((it + 2 * kst) * 2 * 64 + lane) * 8;
        *(fd_short8*)f = hi;
        *(fd_short8*)(f + 64 * 8) = lo;
      }
      // read-out of the memory before the chunk: O = a^{i+1} Q S
      fd_float4 acc[4];
#pragma unroll
      for (int it = 0; it < 4; ++it) acc[it] = fd_float4{0, 0, 0, 0};
#pragma unroll
      for (int ns = 0; ns < NP / 32; ++ns) {
        float x[8];
#pragma unroll
        for (int e = 0; e < 8; ++e) x[e] = S[2 * ns + (e >> 2)][e & 3];
        fd_short8 hi, lo;
        split_pair(x, hi, lo);
#pragma unroll
        for (int it = 0; it < 4; ++it) {
          const int n = ns * 32 + 4 * g4;
          const fd_short8 aa =
              fd_join(*(const fd_short4*)(qs + fd_row<NP>(it, l16, n)),
                      *(const fd_short4*)(qs + fd_row<NP>(it, l16, n + 16)));
          acc[it] = mfma_bf16(aa, hi, acc[it]);
          acc[it] = mfma_bf16(aa, lo, acc[it]);
        }
      }
#pragma unroll
      for (int it = 0; it < 4; ++it)
#pragma unroll
        for (int r = 0; r < 4; ++r)
          acc[it][r] *= pw[it * 16 + g4 * 4 + r + 1];
      __syncthreads();     // score fragments
      fd_short8 vb[2];
#pragma unroll
      for (int kst = 0; kst < 2; ++kst)
        vb[kst] = fd_join(
            *(const fd_short4*)(vt + fd_swz(wave, l16, kst * 32 + 4 * g4)),
            *(const fd_short4*)(vt + fd_swz(wave, l16,
                                            kst * 32 + 16 + 4 * g4)));
#pragma unroll
      for (int it = 0; it < 4; ++it)
#pragma unroll
        for (int kst = 0; kst < 2; ++kst) {
          if (kst * 32 > it * 16 + 15) continue;
          const uint16_t* f = af + ((it + 2 * kst) * 2 * 64 + lane) * 8;
          acc[it] = mfma_bf16(*(const fd_short8*)f, vb[kst], acc[it]);
          acc[it] = mfma_bf16(*(const fd_short8*)(f + 64 * 8), vb[kst],
                              acc[it]);
        }
      if (pc < P) {
        // uniform row base + one 32-bit lane offset
        const int off = g4 * 4 * H * P + pc;
        const int full = L == FD_C ? FD_C : L - g4 * 4;
#pragma unroll
        for (int it = 0; it < 4; ++it)
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            float* o = out + ((int64_t)(c0 + it * 16 + r) * H + h) * P;
            if (it * 16 + r < full) o[off] = acc[it][r];
          }
      }
    }
    // two eight-wave workgroups share a compute unit and its registers: the
    // next rows are requested when the read-out's registers are free
    if (NW == 8 && c0 + FD_C < row1) fetch(c0 + FD_C);
    // memory after the chunk
    const float aL = pw[L];
#pragma unroll
    for (int nt = 0; nt < NTILE; ++nt) S[nt] *= aL;
#pragma unroll
    for (int js = 0; js < 2; ++js) {
      const fd_short8 raw = *(const fd_short8*)(
          vt + fd_swz(wave, l16, js * 32 + g4 * 8));
      // a^{L-1-j}; zero past the last row
      float x[8];
      const float* pl = pw + L - 1 - js * 32 - g4 * 8;
#pragma unroll
      for (int e = 0; e < 8; ++e)
        x[e] = bf16_to_f32((uint16_t)raw[e]) * pl[-e];
      fd_short8 hi, lo;
      split_pair(x, hi, lo);
#pragma unroll
      for (int nt = 0; nt < NTILE; ++nt) {
        const fd_short8 aa = *(const fd_short8*)(
            kt + fd_swz(nt, l16, js * 32 + g4 * 8));
        S[nt] = mfma_bf16(aa, hi, S[nt]);
        S[nt] = mfma_bf16(aa, lo, S[nt]);
      }
    }
    __syncthreads();       // the staged rows are free again
  }
  float* dst = STATE_ONLY ? wk : (last && wk == nullptr ? st : nullptr);
  if (dst != nullptr && pc < P) {
#pragma unroll
    for (int nt = 0; nt < NTILE; ++nt)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int n = nt * 16 + g4 * 4 + r;
        if (n < N) dst[(int64_t)n * P + pc] = S[nt][r];
      }
  }
}

// work[segment] holds the segment's own contribution; becomes the memory at
// the segment's start, in order, and the slot gets the final one.
// seg_first[i] .. seg_first[i + 1] are the segments of the i-th sequence.
__global__ __launch_bounds__(256) void fixed_decay_carry_kernel(
    float* __restrict__ work, float* __restrict__ state,
    const float* __restrict__ decay, const int32_t* __restrict__ segs,
    int nseg, const int32_t* __restrict__ seg_first,
    const int32_t* __restrict__ seq_start,
    const int32_t* __restrict__ seq_slots, int H, int64_t NP_) {
  const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (i >= NP_) return;
  const int h = blockIdx.y;
  const int s0 = seg_first[blockIdx.z], s1 = seg_first[blockIdx.z + 1];
  if (s0 == s1) return;
  const int seq = segs[2 * nseg + s0];
  const float a = decay[h];
  float* st = state + ((int64_t)seq_slots[seq] * H + h) * NP_ + i;
  float x = seq_start[seq] == 0 ? 0.0f : *st;
  for (int s = s0; s < s1; ++s) {
    float* w = work + ((int64_t)s * H + h) * NP_ + i;
    const float own = *w;
    *w = x;
    x = powf(a, (float)(segs[nseg + s] - segs[s])) * x + own;
  }
  *st = x;
}

// ---------------------------------------------------------------------------
int64_t fixed_decay_chunk_keys() { return 128; }   // widest N of the chunks

static void fd_check(const torch::Tensor& out, const torch::Tensor& q,
                     const torch::Tensor& k, const torch::Tensor& v,
                     const torch::Tensor& decay, const torch::Tensor& state) {
  TORCH_CHECK(v.is_cuda() && v.dim() == 3 && v.stride(2) == 1 &&
              q.dim() == 3 && q.stride(2) == 1 && k.dim() == 3 &&
              k.stride(2) == 1 && q.dtype() == v.dtype() &&
              k.dtype() == v.dtype() && q.sizes() == k.sizes() &&
              q.size(0) == v.size(0));
  const int64_t T = v.size(0), H = v.size(1), P = v.size(2);
  const int64_t G = q.size(1), N = q.size(2);
  TORCH_CHECK(G >= 1 && H % G == 0 && N >= 1 && P >= 1);
  TORCH_CHECK(out.dtype() == torch::kFloat32 && out.is_contiguous() &&
              out.numel() == T * H * P);
  TORCH_CHECK(decay.dtype() == torch::kFloat32 && decay.is_contiguous() &&
              decay.numel() == H);
  TORCH_CHECK(state.dtype() == torch::kFloat32 && state.is_contiguous() &&
              state.dim() == 2 && state.size(1) == H * N * P,
              "memory slot width must be heads * keys * values");
}

static void fd_check_seqs(const torch::Tensor& seq_start,
                          const torch::Tensor& seq_slots) {
  TORCH_CHECK(seq_start.dtype() == torch::kInt32 &&
              seq_slots.dtype() == torch::kInt32 &&
              seq_start.is_contiguous() && seq_slots.is_contiguous() &&
              seq_start.numel() == seq_slots.numel());
}

void fixed_decay_step(torch::Tensor out, torch::Tensor q, torch::Tensor k,
                      torch::Tensor v, torch::Tensor decay,
                      torch::Tensor state, torch::Tensor seqs,
                      torch::Tensor seq_cu, torch::Tensor seq_start,
                      torch::Tensor seq_slots, bool silu) {
  fd_check(out, q, k, v, decay, state);
  fd_check_seqs(seq_start, seq_slots);
  const int H = v.size(1), P = v.size(2), G = q.size(1), N = q.size(2);
  const int S = seqs.numel();
  TORCH_CHECK(seqs.dtype() == torch::kInt32 && seqs.is_contiguous() &&
              seq_cu.dtype() == torch::kInt32 &&
              seq_cu.numel() == seq_start.numel() + 1);
  TORCH_CHECK(N <= 512, "key width above 512 is not supported");
  if (v.size(0) == 0 || S == 0) return;
  hipStream_t stream = at::cuda::getCurrentCUDAStream();
  const dim3 grid((P + FD_PT - 1) / FD_PT, H, S);
  const size_t shmem =
      sizeof(float) * (2 * (size_t)FD_ROWS * N + FD_ROWS * FD_PT +
                       2 * 4 * FD_PT);
  const bool v4 = P % 4 == 0 &&
                  reinterpret_cast<uintptr_t>(state.data_ptr()) % 16 == 0;
#define FD_STEP(NPERV, V4V)                                                   \
  do {                                                                        \
    auto kern = fixed_decay_step_kernel<act_t, NPERV, V4V>;                   \
    if (shmem > 64 * 1024)                                                    \
      (void)hipFuncSetAttribute((const void*)kern,                            \
                                hipFuncAttributeMaxDynamicSharedMemorySize,   \
                                (int)shmem);                                  \
    hipLaunchKernelGGL(                                                       \
        kern, grid, dim3(256), shmem, stream, (float*)out.data_ptr(),         \
        (const act_t*)q.data_ptr(), (int64_t)q.stride(0),                     \
        (int64_t)q.stride(1), (const act_t*)k.data_ptr(),                     \
        (int64_t)k.stride(0), (int64_t)k.stride(1),                           \
        (const act_t*)v.data_ptr(), (int64_t)v.stride(0),                     \
        (int64_t)v.stride(1), (const float*)decay.data_ptr(),                 \
        (float*)state.data_ptr(), (const int32_t*)seqs.data_ptr(),            \
        (const int32_t*)seq_cu.data_ptr(),                                    \
        (const int32_t*)seq_start.data_ptr(),                                 \
        (const int32_t*)seq_slots.data_ptr(), H, G, N, P, silu ? 1 : 0);      \
  } while (0)
#define FD_STEP_N(NPERV)                                                      \
  do {                                                                        \
    if (v4) FD_STEP(NPERV, true);                                             \
    else FD_STEP(NPERV, false);                                               \
  } while (0)
  IGW_DISPATCH_ACT(v, {
    if (N <= 16) FD_STEP_N(1);
    else if (N <= 32) FD_STEP_N(2);
    else if (N <= 64) FD_STEP_N(4);
    else if (N <= 128) FD_STEP_N(8);
    else if (N <= 256) FD_STEP_N(16);
    else FD_STEP_N(32);
  });
#undef FD_STEP_N
#undef FD_STEP
  (void)hipGetLastError();   // a refused attribute must not poison the check
  HIP_CHECK_KERNEL();
}

// segs int32 [5, nseg] (see the kernel); work fp32 [nseg, H, N, P] when the
// prompts are cut into segments that run side by side, with seg_first int32
// [sequences + 1]; without work every sequence is one segment.
void fixed_decay_chunks(torch::Tensor out, torch::Tensor q, torch::Tensor k,
                        torch::Tensor v, torch::Tensor decay,
                        torch::Tensor state, torch::Tensor segs,
                        c10::optional<torch::Tensor> work,
                        c10::optional<torch::Tensor> seg_first,
                        torch::Tensor seq_start, torch::Tensor seq_slots,
                        bool silu) {
  fd_check(out, q, k, v, decay, state);
  fd_check_seqs(seq_start, seq_slots);
  const int H = v.size(1), P = v.size(2), G = q.size(1), N = q.size(2);
  TORCH_CHECK(v.scalar_type() == torch::kBFloat16 &&
              N <= fixed_decay_chunk_keys());
  TORCH_CHECK(segs.dtype() == torch::kInt32 && segs.is_contiguous() &&
              segs.dim() == 2 && segs.size(0) == 5);
  const int nseg = segs.size(1);
  TORCH_CHECK(work.has_value() == seg_first.has_value());
  if (work.has_value())
    TORCH_CHECK(work->dtype() == torch::kFloat32 && work->is_contiguous() &&
                work->numel() == (int64_t)nseg * H * N * P &&
                seg_first->dtype() == torch::kInt32 &&
                seg_first->is_contiguous());
  if (v.size(0) == 0 || nseg == 0) return;
  hipStream_t stream = at::cuda::getCurrentCUDAStream();
  const int nw = P <= 64 ? 4 : 8;
  const dim3 grid((P + nw * 16 - 1) / (nw * 16), H, nseg);
  auto aligned = [](const torch::Tensor& t) {
    return reinterpret_cast<uintptr_t>(t.data_ptr()) % 16 == 0 &&
           t.stride(0) % 8 == 0 && t.stride(1) % 8 == 0;
  };
  const bool vec = N % 8 == 0 && P % 8 == 0 && aligned(q) && aligned(k) &&
                   aligned(v);
#define FD_CHUNK(NPV, NWV, VECV, SOV)                                         \
  hipLaunchKernelGGL(                                                         \
      (fixed_decay_chunk_kernel<NPV, NWV, VECV, SOV>), grid, dim3(NWV * 64),  \
      0, stream, (float*)out.data_ptr(), (const uint16_t*)q.data_ptr(),       \
      (int64_t)q.stride(0), (int64_t)q.stride(1),                             \
      (const uint16_t*)k.data_ptr(), (int64_t)k.stride(0),                    \
      (int64_t)k.stride(1), (const uint16_t*)v.data_ptr(),                    \
      (int64_t)v.stride(0), (int64_t)v.stride(1),                             \
      (const float*)decay.data_ptr(), (float*)state.data_ptr(),               \
      work.has_value() ? (float*)work->data_ptr() : nullptr,                  \
      (const int32_t*)segs.data_ptr(), nseg,                                  \
      (const int32_t*)seq_start.data_ptr(),                                   \
      (const int32_t*)seq_slots.data_ptr(), H, G, N, P, silu ? 1 : 0)
#define FD_CHUNK_V(NPV, NWV, SOV)                                             \
  do {                                                                        \
    if (vec) FD_CHUNK(NPV, NWV, true, SOV);                                   \
    else FD_CHUNK(NPV, NWV, false, SOV);                                      \
  } while (0)
#define FD_CHUNK_N(NPV, SOV)                                                  \
  do {                                                                        \
    if (nw == 4) FD_CHUNK_V(NPV, 4, SOV);                                     \
    else FD_CHUNK_V(NPV, 8, SOV);                                             \
  } while (0)
#define FD_CHUNK_ALL(SOV)                                                     \
  do {                                                                        \
    if (N <= 32) FD_CHUNK_N(32, SOV);                                         \
    else if (N <= 64) FD_CHUNK_N(64, SOV);                                    \
    else FD_CHUNK_N(128, SOV);                                                \
  } while (0)
  if (work.has_value()) {
    FD_CHUNK_ALL(true);
    HIP_CHECK_KERNEL();
    const int64_t np = (int64_t)N * P;
    hipLaunchKernelGGL(
        fixed_decay_carry_kernel,
        dim3((unsigned)((np + 255) / 256), H, seg_first->numel() - 1),
        dim3(256), 0, stream, (float*)work->data_ptr(),
        (float*)state.data_ptr(), (const float*)decay.data_ptr(),
        (const int32_t*)segs.data_ptr(), nseg,
        (const int32_t*)seg_first->data_ptr(),
        (const int32_t*)seq_start.data_ptr(),
        (const int32_t*)seq_slots.data_ptr(), H, np);
    HIP_CHECK_KERNEL();
  }
  FD_CHUNK_ALL(false);
#undef FD_CHUNK_ALL
#undef FD_CHUNK_N
#undef FD_CHUNK_V
#undef FD_CHUNK
  HIP_CHECK_KERNEL();
}

}  // namespace igw
