// Linear attention with a decay per head, fixed or formed from every token, over the ragged batch of a
// step, state in 32-bit per sequence slot.
//
// Per head, with q_t, k_t (dim values) and v_t (vdim values) the silu of their projections:
//   S_t = decay S_(t-1) + k_t v_t^T        (dim x vdim),      o_t = S_t^T q_t.
// The heads of a token side by side are then RMS-normed with a gain vector, multiplied by the
// sigmoid of a gate projection and rounded once (`gated_rmsnorm_kernel`).  q | k | v | gate arrive as
// one 32-bit row per token; state, decays, products and sums are 32-bit throughout.
//
// `lightning_scan_kernel`: a workgroup owns (sequence, head, 64 value columns) and walks the
// sequence's new tokens in order; its 256 threads are 4 slices of the key dimension times 64
// columns, a thread keeping its slice of its column of S in registers.  Decode steps and short
// portions use it alone.
//
// Prompts: the tokens of a sequence are cut into chunks of MF_LA_CHUNK.  Unrolling the recurrence
// inside a chunk that starts at token c0 from the state S_in,
//   o_t = decay^(t - c0 + 1) S_in^T q_t + sum_{c0 <= s <= t} decay^(t - s) (q_t . k_s) v_s,
//   S_out = decay^n S_in + sum_s decay^(c0 + n - 1 - s) k_s v_s^T,
// so pass 1 reduces every chunk to its own sum B_c (all chunks side by side), pass 2 folds
// S_in(c + 1) = decay^n S_in(c) + B_c along each sequence, and pass 3 writes every chunk's outputs
// from its S_in and its own tokens (all chunks side by side again).  The order of a position's
// additions depends on where the chunk edges fall inside the step, never on the batch.
//
// The kernels come in three kinds.  MF_LA_SILU is the above.  MF_LA_PLAIN takes q, k and v as projected, times a
// scale each for q and k, and rotates q and k in halves by the token's angles (the sequential kernel on the way
// into LDS; in front of the chunked passes `la_rotate_kernel` turns the rows in place).  MF_LA_MEMORY is a matrix
// memory with exponential gates: with the capped log gates i = cap tanh(zi / cap) and
// f = logsigmoid(cap tanh(zf / cap)) of a token and a running maximum m that starts at 0,
//   m_t = max(f + m_(t-1), i),  S_t = exp(f + m_(t-1) - m_t) S_(t-1) + exp(i - m_t) k_t v_t^T,  n_t likewise with k
// alone; the kernels leave S_t^T q_t, n_t . q_t and exp(-m_t), and what follows divides.  A slot's state holds
// S [H][D][V], then n [H][D], then m [H][column blocks]: the workgroups of a head's column blocks all walk m, each
// from and into a copy of its own, since one may end before another begins.  In the chunked form `memory_gates_kernel` first walks m along every
// sequence (a scan over (f, i) pairs under m -> max(m + f, i)), and leaves for every token the sum since its
// chunk's start of the logarithms of the factors on S (in double: differences of two of them weigh the pairs
// of tokens inside the chunk), the logarithm of its own weight, and exp(-m_t).
#include "common.h"

#define MF_LA_CHUNK 64
#define MF_LA_TT 8     // tokens whose q and k are staged together in the sequential kernel

#define MF_LA_SILU 0
#define MF_LA_PLAIN 1
#define MF_LA_MEMORY 2

// what a token's gates come to in the chunked form of the matrix memory
struct MemoryGate {
  double decay_log;      // sum since the chunk's start, this token included, of the logarithms of the factors on S
  float take_log;        // logarithm of the weight of the token's own k v^T
  float floor;           // exp(-m)
};

// what the kinds other than MF_LA_SILU need besides
struct LaExtra {
  float q_scale, k_scale;
  const float* cos_t;    // rotation in halves of q and k, tables [positions][rot / 2]; rot 0: none
  const float* sin_t;
  const int* positions;
  int rot;
  int off_i, off_f;      // columns of the gates' projections in a row (MF_LA_MEMORY)
  float cap;
  float* den;            // [tokens][H]: n_t . q_t
  float* floor;          // [tokens][H]: exp(-m_t)
  const MemoryGate* gates;   // [tokens][H], chunked form
  const float* chunk_decay;  // [chunks][H]
  float* n_ws;               // [chunks][H][D]: the chunk's own sum of n, then the n it starts from
};

__device__ __forceinline__ float la_sigmoid(float x) { return 1.0f / (1.0f + expf(-x)); }
__device__ __forceinline__ float la_silu(float x) { return x * la_sigmoid(x); }
__device__ __forceinline__ float la_log_sigmoid(float x) { return fminf(x, 0.f) - log1pf(expf(-fabsf(x))); }
__device__ __forceinline__ float la_cap(float x, float cap) { return cap * tanhf(x / cap); }

// copies of m a head keeps: one per block of 64 value columns
__host__ __device__ __forceinline__ int la_m_copies(int V) { return (V + 63) / 64; }

// floats of a slot's state
template <int KIND>
__device__ __forceinline__ size_t la_state_len(int H, int D, int V) {
  return KIND == MF_LA_MEMORY ? (size_t)H * ((size_t)D * V + D + la_m_copies(V)) : (size_t)H * D * V;
}

// value d of head `hd` of a row's q or k part: rotated in halves by the token's angles where it is to be
__device__ __forceinline__ float la_rotated(const float* __restrict__ head, int d, int rot, const float* __restrict__ cs,
                                            const float* __restrict__ sn) {
  const float x = head[d];
  if (d >= rot) return x;
  const int half = rot / 2;
  return d < half ? x * cs[d] - head[d + half] * sn[d] : x * cs[d - half] + head[d - half] * sn[d - half];
}

// proj row: q [H D] | k [H D] | v [H V] | gate [H V]
// DS registers of a thread: its slice of the key dimension (dim <= 4 DS)
template <int DS, int KIND>
__global__ __launch_bounds__(256) void lightning_scan_kernel(const float* __restrict__ proj, int row_len,
                                                             const int* __restrict__ cu_seqlens,
                                                             const int* __restrict__ slot_ids,
                                                             const float* __restrict__ decays,
                                                             float* __restrict__ state, float* __restrict__ out,
                                                             int H, int D, int V, LaExtra ex) {
  __shared__ float sq[MF_LA_TT][4 * DS], sk[MF_LA_TT][4 * DS];
  __shared__ float partial[MF_LA_TT][4][64];
  __shared__ float s_i[MF_LA_TT], s_f[MF_LA_TT], s_keep[MF_LA_TT], s_take[MF_LA_TT], s_floor[MF_LA_TT];
  __shared__ float den_part[MF_LA_TT][4];
  const int seq = blockIdx.x, h = blockIdx.y;
  const int col = blockIdx.z * 64 + (threadIdx.x & 63), slice = threadIdx.x >> 6;
  const bool live = col < V;
  const int t0 = cu_seqlens[seq], t1 = cu_seqlens[seq + 1];
  const float decay = KIND == MF_LA_MEMORY ? 1.f : decays[h];
  float* slot = state + (size_t)slot_ids[seq] * la_state_len<KIND>(H, D, V);
  float* st = slot + ((size_t)h * D) * V + col;
  float* st_n = slot + (size_t)H * D * V + (size_t)h * D;
  float* st_m = slot + (size_t)H * D * V + (size_t)H * D + (size_t)h * la_m_copies(V) + blockIdx.z;
  // n: lane l of a wave keeps value slice DS + l (the workgroup of the first columns alone); m: thread 0 alone
  const int lane = threadIdx.x & 63;
  const int dn = slice * DS + lane;
  const bool has_n = KIND == MF_LA_MEMORY && blockIdx.z == 0 && lane < DS && dn < D;
  float nn = has_n ? st_n[dn] : 0.f;
  float m = KIND == MF_LA_MEMORY && threadIdx.x == 0 ? *st_m : 0.f;
  float S[DS];
#pragma unroll
  for (int i = 0; i < DS; ++i) {
    const int d = slice * DS + i;
    S[i] = (live && d < D) ? st[(size_t)d * V] : 0.f;
  }
  const int off_k = H * D, off_v = 2 * H * D;
  for (int tb = t0; tb < t1; tb += MF_LA_TT) {
    const int nt = min(MF_LA_TT, t1 - tb);
    __syncthreads();
    for (int i = threadIdx.x; i < nt * 4 * DS; i += 256) {
      const int tt = i / (4 * DS), d = i % (4 * DS);
      const float* row = proj + (size_t)(tb + tt) * row_len + h * D;
      float qv = 0.f, kv = 0.f;
      if (d < D) {
        if (KIND == MF_LA_SILU) {
          qv = la_silu(row[d]);
          kv = la_silu(row[off_k + d]);
        } else if (KIND == MF_LA_PLAIN && d < ex.rot) {
          const size_t at = (size_t)ex.positions[tb + tt] * (ex.rot / 2);
          qv = la_rotated(row, d, ex.rot, ex.cos_t + at, ex.sin_t + at) * ex.q_scale;
          kv = la_rotated(row + off_k, d, ex.rot, ex.cos_t + at, ex.sin_t + at) * ex.k_scale;
        } else {
          qv = row[d] * ex.q_scale;
          kv = row[off_k + d] * ex.k_scale;
        }
      }
      sq[tt][d] = qv;
      sk[tt][d] = kv;
    }
    if (KIND == MF_LA_MEMORY) {
      if (threadIdx.x < nt) {
        const float* row = proj + (size_t)(tb + threadIdx.x) * row_len;
        s_i[threadIdx.x] = la_cap(row[ex.off_i + h], ex.cap);
        s_f[threadIdx.x] = la_log_sigmoid(la_cap(row[ex.off_f + h], ex.cap));
      }
      __syncthreads();
      if (threadIdx.x == 0)
        for (int tt = 0; tt < nt; ++tt) {
          const float carried = s_f[tt] + m, mine = s_i[tt];
          m = fmaxf(carried, mine);
          s_keep[tt] = expf(carried - m);
          s_take[tt] = expf(mine - m);
          s_floor[tt] = expf(-m);
        }
    }
    __syncthreads();
    for (int tt = 0; tt < nt; ++tt) {
      float vv = live ? proj[(size_t)(tb + tt) * row_len + off_v + h * V + col] : 0.f;
      if (KIND == MF_LA_SILU) vv = la_silu(vv);
      float keep = decay;
      if (KIND == MF_LA_MEMORY) {
        keep = s_keep[tt];
        vv *= s_take[tt];
        if (blockIdx.z == 0) {
          nn = has_n ? fmaf(keep, nn, s_take[tt] * sk[tt][dn]) : 0.f;
          const float part = wave_sum(has_n ? nn * sq[tt][dn] : 0.f);
          if (lane == 0) den_part[tt][slice] = part;
        }
      }
      float o = 0.f;
#pragma unroll
      for (int i = 0; i < DS; ++i) {
        const int d = slice * DS + i;
        S[i] = fmaf(keep, S[i], sk[tt][d] * vv);
        o = fmaf(S[i], sq[tt][d], o);
      }
      partial[tt][slice][threadIdx.x & 63] = o;
    }
    __syncthreads();
    for (int i = threadIdx.x; i < nt * 64; i += 256) {
      const int tt = i >> 6, c = i & 63;
      const int cc = blockIdx.z * 64 + c;
      if (cc < V)
        out[(size_t)(tb + tt) * H * V + h * V + cc] =
            ((partial[tt][0][c] + partial[tt][1][c]) + partial[tt][2][c]) + partial[tt][3][c];
    }
    if (KIND == MF_LA_MEMORY && blockIdx.z == 0 && threadIdx.x < nt) {
      const int tt = threadIdx.x;
      ex.den[(size_t)(tb + tt) * H + h] = ((den_part[tt][0] + den_part[tt][1]) + den_part[tt][2]) + den_part[tt][3];
      ex.floor[(size_t)(tb + tt) * H + h] = s_floor[tt];
    }
  }
  if (live) {
#pragma unroll
    for (int i = 0; i < DS; ++i) {
      const int d = slice * DS + i;
      if (d < D) st[(size_t)d * V] = S[i];
    }
  }
  if (KIND == MF_LA_MEMORY) {
    if (has_n) st_n[dn] = nn;
    if (threadIdx.x == 0) *st_m = m;
  }
}

// the rotation in halves of the first `n_heads` heads of D values of every row, in place
__global__ __launch_bounds__(256) void la_rotate_kernel(float* __restrict__ rows, int row_len, const float* __restrict__ cos_t,
                                                        const float* __restrict__ sin_t, const int* __restrict__ positions,
                                                        int n_heads, int D, int rot) {
  const int t = blockIdx.x, half = rot / 2;
  const float* cs = cos_t + (size_t)positions[t] * half;
  const float* sn = sin_t + (size_t)positions[t] * half;
  for (int i = threadIdx.x; i < n_heads * half; i += 256) {
    const int e = i % half;
    float* a = rows + (size_t)t * row_len + (size_t)(i / half) * D + e;
    const float x = a[0], z = a[half];
    a[0] = x * cs[e] - z * sn[e];
    a[half] = z * cs[e] + x * sn[e];
  }
}

// The running maximum of the matrix memory along every sequence and what follows from it.  A workgroup owns
// (sequence, head); its 16 waves take 16 chunks of 64 tokens a round.
#define MF_LA_GATE_WAVES 16
__global__ __launch_bounds__(64 * MF_LA_GATE_WAVES) void memory_gates_kernel(
    const float* __restrict__ proj, int row_len, const int* __restrict__ cu_seqlens, const int* __restrict__ slot_ids,
    const int* __restrict__ seq_first_chunk, float* __restrict__ state, MemoryGate* __restrict__ gates,
    float* __restrict__ chunk_decay, int H, int D, int V, int off_i, int off_f, float cap) {
  __shared__ float wave_a[MF_LA_GATE_WAVES], wave_b[MF_LA_GATE_WAVES];
  const int seq = blockIdx.x, h = blockIdx.y;
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6;
  const int t0 = cu_seqlens[seq], t1 = cu_seqlens[seq + 1];
  const int copies = la_m_copies(V);
  float* st_m = state + (size_t)slot_ids[seq] * la_state_len<MF_LA_MEMORY>(H, D, V) + (size_t)H * D * V + (size_t)H * D +
                (size_t)h * copies;
  float m = *st_m;                 // the maximum before the round's first token
  for (int base = t0; base < t1; base += 64 * MF_LA_GATE_WAVES) {
    const int t = base + threadIdx.x;
    const bool live = t < t1;
    float f = 0.f, i = -INFINITY;  // (a token beyond the sequence leaves m as it is)
    if (live) {
      const float* row = proj + (size_t)t * row_len;
      i = la_cap(row[off_i + h], cap);
      f = la_log_sigmoid(la_cap(row[off_f + h], cap));
    }
    // inclusive scan: the wave's tokens up to this one take m to max(m + a, b)
    float a = f, b = i;
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const float pa = __shfl_up(a, o, MF_WAVE), pb = __shfl_up(b, o, MF_WAVE);
      if (lane >= o) {
        b = fmaxf(pb + a, b);
        a = pa + a;
      }
    }
    __syncthreads();
    if (lane == 63) { wave_a[w] = a; wave_b[w] = b; }
    __syncthreads();
    float m_in = m;
    for (int k = 0; k < MF_LA_GATE_WAVES; ++k) {
      if (k == w) m_in = m;
      m = fmaxf(m + wave_a[k], wave_b[k]);
    }
    const float mt = fmaxf(m_in + a, b);
    float before = __shfl_up(mt, 1, MF_WAVE);
    if (lane == 0) before = m_in;
    double L = live ? (double)(f + before - mt) : 0.0;
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const double p = __shfl_up(L, o, MF_WAVE);
      if (lane >= o) L += p;
    }
    if (live) {
      MemoryGate g;
      g.decay_log = L;
      g.take_log = i - mt;
      g.floor = expf(-mt);
      gates[(size_t)t * H + h] = g;
    }
    if (lane == 63 && base + 64 * w < t1)
      chunk_decay[(size_t)(seq_first_chunk[seq] + (base - t0) / 64 + w) * H + h] = expf((float)L);
  }
  if (threadIdx.x < copies) st_m[threadIdx.x] = m;
}
static_assert(MF_LA_CHUNK == 64, "a wave of memory_gates_kernel takes a chunk");

// ------------------------------------------------------------------ the chunked form
// chunk table: int32 [2][n_chunks] = first token, tokens; then [n_seqs + 1] first chunks of the sequences
//
// The products of the chunked form run on the matrix cores in 32-bit (16x16x4 MFMA with float operands: the
// same multiply-adds as the plain form, no rounding of an operand): a lane gives A[i = lane % 16][k = lane / 16]
// and B[k = lane / 16][j = lane % 16] and holds D[i = 4 (lane / 16) + r][j = lane % 16], r < 4.  Operands are
// staged in LDS with rows 4 floats longer than they are, which spreads a fragment's 64 reads over the banks.
#define MF_LA_VS (64 + 4)     // row stride of tiles of 64 columns

// Staging of a [MF_LA_CHUNK][W] tile of 32-bit rows into LDS, silu applied or not: rows tt >= n and
// columns beyond `valid` are zero.  With `vec` (every row start and `valid` multiples of 4 floats) a thread's
// loads are 16 bytes each and all issued before the first is used.
template <int WP, bool SILU>
__device__ __forceinline__ void stage_tile(float* __restrict__ dst, int dst_stride, const float* __restrict__ src,
                                           size_t src_stride, int n_rows, int n, int valid, bool vec,
                                           float scale = 1.0f) {
  constexpr int W4 = WP / 4;
  if (vec) {
    for (int base = 0; base < n_rows * W4; base += 256 * 8) {
      float4 tmp[8];
#pragma unroll
      for (int u = 0; u < 8; ++u) {
        const int i = base + u * 256 + threadIdx.x;
        const int tt = i / W4, c4 = (i % W4) * 4;
        tmp[u] = (i < n_rows * W4 && tt < n && c4 < valid) ? *(const float4*)(src + (size_t)tt * src_stride + c4)
                                                             : float4{0.f, 0.f, 0.f, 0.f};
      }
#pragma unroll
      for (int u = 0; u < 8; ++u) {
        const int i = base + u * 256 + threadIdx.x;
        if (i >= n_rows * W4) continue;
        const int tt = i / W4, c4 = (i % W4) * 4;
        float4 v = tmp[u];
        if (SILU) { v.x = la_silu(v.x); v.y = la_silu(v.y); v.z = la_silu(v.z); v.w = la_silu(v.w); }
        else { v.x *= scale; v.y *= scale; v.z *= scale; v.w *= scale; }
        *(float4*)(dst + tt * dst_stride + c4) = v;
      }
    }
  } else {
    for (int i = threadIdx.x; i < n_rows * WP; i += 256) {
      const int tt = i / WP, cc = i % WP;
      const float v = (tt < n && cc < valid) ? src[(size_t)tt * src_stride + cc] : 0.f;
      dst[tt * dst_stride + cc] = SILU ? la_silu(v) : v * scale;
    }
  }
}

// pass 1: B_c[d][v] = sum_s decay^(n - 1 - s) k_s[d] v_s[v] = K'^T V; a workgroup owns (chunk, head, 64
// columns), a wave 16 of the columns.
template <int DS, int KIND>
__global__ __launch_bounds__(256) void lightning_chunk_sum_kernel(const float* __restrict__ proj, int row_len,
                                                                  const int* __restrict__ chunk_t0,
                                                                  const int* __restrict__ chunk_n,
                                                                  const float* __restrict__ decays,
                                                                  float* __restrict__ bsum, int H, int D, int V,
                                                                  LaExtra ex) {
  constexpr int DP = 4 * DS, DPS = DP + 4;
  constexpr bool SILU = KIND == MF_LA_SILU;
  extern __shared__ float lds[];
  float* sk = lds;                          // [CHUNK][DPS]
  float* sv = sk + MF_LA_CHUNK * DPS;       // [CHUNK][VS]
  const int c = blockIdx.x, h = blockIdx.y, v0 = blockIdx.z * 64;
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6;
  const int t0 = chunk_t0[c], n = chunk_n[c];
  const float decay = KIND == MF_LA_MEMORY ? 1.f : decays[h];
  const int off_k = H * D, off_v = 2 * H * D;
  const bool vec = D % 4 == 0 && V % 4 == 0 && row_len % 4 == 0;
  const float* rows = proj + (size_t)t0 * row_len;
  stage_tile<DP, SILU>(sk, DPS, rows + off_k + h * D, row_len, MF_LA_CHUNK, n, D, vec, SILU ? 1.f : ex.k_scale);
  stage_tile<64, SILU>(sv, MF_LA_VS, rows + off_v + h * V + v0, row_len, MF_LA_CHUNK, n, min(64, V - v0), vec);
  __shared__ float to_end[MF_LA_CHUNK];          // decay^(n - 1 - s): what a token's k v^T is worth at the chunk's end
  if (threadIdx.x < MF_LA_CHUNK) {
    float x = 0.f;
    if (threadIdx.x < n) {
      if (KIND == MF_LA_MEMORY) {
        const MemoryGate mine = ex.gates[(size_t)(t0 + threadIdx.x) * H + h];
        x = expf((float)(ex.gates[(size_t)(t0 + n - 1) * H + h].decay_log - mine.decay_log) + mine.take_log);
      } else {
        x = powf(decay, (float)(n - 1 - threadIdx.x));
      }
    }
    to_end[threadIdx.x] = x;
  }
  __syncthreads();
  if (KIND == MF_LA_MEMORY && blockIdx.z == 0)
    for (int d = threadIdx.x; d < D; d += 256) {
      float a = 0.f;
      for (int s = 0; s < n; ++s) a = fmaf(to_end[s], sk[s * DPS + d], a);
      ex.n_ws[((size_t)c * H + h) * D + d] = a;
    }
  const int col = lane & 15, g = lane >> 4;
  for (int di = 0; di < DP / 16; ++di) {
    floatx4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
    for (int kk = 0; kk < MF_LA_CHUNK / 4; ++kk) {
      const int srow = 4 * kk + g;
      acc = __builtin_amdgcn_mfma_f32_16x16x4f32(sk[srow * DPS + 16 * di + col] * to_end[srow], sv[srow * MF_LA_VS + 16 * w + col], acc,
                                                 0, 0, 0);
    }
    const int cc = v0 + 16 * w + col;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int dd = 16 * di + 4 * g + r;
      if (dd < D && cc < V) bsum[(((size_t)c * H + h) * D + dd) * V + cc] = acc[r];
    }
  }
}

// pass 2: along each sequence, S_in(first) = stored state, S_in(c + 1) = decay^n(c) S_in(c) + B_c, the
// last one stored back as the sequence's state.  B_c is replaced by S_in(c) in place.  One thread per
// element of the state; grid (sequence, head, elements / 256).
template <int KIND>
__global__ __launch_bounds__(256) void lightning_chunk_fold_kernel(const int* __restrict__ chunk_n,
                                                                   const int* __restrict__ seq_first_chunk,
                                                                   const int* __restrict__ slot_ids,
                                                                   const float* __restrict__ decays,
                                                                   float* __restrict__ bsum, float* __restrict__ state,
                                                                   int H, int D, int V, LaExtra ex) {
  const int seq = blockIdx.x, h = blockIdx.y;
  const int DV = D * V;
  const int e = blockIdx.z * 256 + threadIdx.x;
  const bool is_n = KIND == MF_LA_MEMORY && e >= DV;        // behind S, the values of n
  if (e >= DV && !(is_n && e < DV + D)) return;
  const int c0 = seq_first_chunk[seq], c1 = seq_first_chunk[seq + 1];
  const float decay = KIND == MF_LA_MEMORY ? 1.f : decays[h];
  float* slot = state + (size_t)slot_ids[seq] * la_state_len<KIND>(H, D, V);
  float* st = is_n ? slot + (size_t)H * DV + (size_t)h * D + (e - DV) : slot + (size_t)h * DV + e;
  float* first = is_n ? ex.n_ws + (size_t)h * D + (e - DV) : bsum + (size_t)h * DV + e;
  const size_t stride = (size_t)H * (is_n ? D : DV);
  const float whole = powf(decay, (float)MF_LA_CHUNK);      // a whole chunk's decay
  float S = *st;
  for (int c = c0; c < c1; ++c) {
    float* b = first + c * stride;
    const float B = *b;
    *b = S;
    S = fmaf(KIND == MF_LA_MEMORY ? ex.chunk_decay[(size_t)c * H + h]
                                     : (chunk_n[c] == MF_LA_CHUNK ? whole : powf(decay, (float)chunk_n[c])),
             S, B);
  }
  *st = S;
}

// pass 3: the outputs of a chunk from S_in and its own tokens.  A workgroup owns (chunk, head, 64 columns).
// First the decayed scores a[t][s] = decay^(t - s) (q_t . k_s), s <= t, tile by tile (the tiles above the
// diagonal are neither formed nor read), then for every 16 tokens x 16 columns
// o = decay^(t + 1) (Q S_in) + a V: the first product's sums are scaled row by row before the second
// product adds onto them.
template <int DS, int KIND>
__global__ __launch_bounds__(256) void lightning_chunk_out_kernel(const float* __restrict__ proj, int row_len,
                                                                  const int* __restrict__ chunk_t0,
                                                                  const int* __restrict__ chunk_n,
                                                                  const float* __restrict__ decays,
                                                                  const float* __restrict__ s_in,
                                                                  float* __restrict__ out, int H, int D, int V,
                                                                  LaExtra ex) {
  constexpr int DP = 4 * DS, DPS = DP + 4;
  constexpr bool SILU = KIND == MF_LA_SILU;
  __shared__ double s_decay[MF_LA_CHUNK];            // the gates' sums of logarithms (MF_LA_MEMORY)
  __shared__ float s_take[MF_LA_CHUNK];
  extern __shared__ float lds[];
  float* sq = lds;                                   // [CHUNK][DPS]
  float* sk = sq + MF_LA_CHUNK * DPS;                 // [CHUNK][DPS]
  float* sa = sk + MF_LA_CHUNK * DPS;                 // [CHUNK][VS]: decayed scores
  float* sv = sa + MF_LA_CHUNK * MF_LA_VS;            // [CHUNK][VS]
  float* ss = sv + MF_LA_CHUNK * MF_LA_VS;            // [DP][VS]: S_in of this head and these columns
  float* dpow = ss + DP * MF_LA_VS;                   // [CHUNK + 1]: decay^i; what S_in is worth after i tokens
  const int c = blockIdx.x, h = blockIdx.y, v0 = blockIdx.z * 64;
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6;
  const int t0 = chunk_t0[c], n = chunk_n[c];
  const float decay = KIND == MF_LA_MEMORY ? 1.f : decays[h];
  const int off_k = H * D, off_v = 2 * H * D;
  const bool vec = D % 4 == 0 && V % 4 == 0 && row_len % 4 == 0;
  const float* rows = proj + (size_t)t0 * row_len;
  stage_tile<DP, SILU>(sq, DPS, rows + h * D, row_len, MF_LA_CHUNK, n, D, vec, SILU ? 1.f : ex.q_scale);
  stage_tile<DP, SILU>(sk, DPS, rows + off_k + h * D, row_len, MF_LA_CHUNK, n, D, vec, SILU ? 1.f : ex.k_scale);
  stage_tile<64, SILU>(sv, MF_LA_VS, rows + off_v + h * V + v0, row_len, MF_LA_CHUNK, n, min(64, V - v0), vec);
  stage_tile<64, false>(ss, MF_LA_VS, s_in + (((size_t)c * H + h) * D) * V + v0, V, DP, D, min(64, V - v0), vec);
  if (KIND == MF_LA_MEMORY) {
    if (threadIdx.x < MF_LA_CHUNK) {
      // (tokens beyond the chunk's weigh nothing: their v is zero, and no output row reads their scores)
      const MemoryGate g = threadIdx.x < n ? ex.gates[(size_t)(t0 + threadIdx.x) * H + h] : MemoryGate{0.0, 0.f, 0.f};
      s_decay[threadIdx.x] = g.decay_log;
      s_take[threadIdx.x] = g.take_log;
      dpow[threadIdx.x + 1] = expf((float)g.decay_log);
    }
  } else if (threadIdx.x <= MF_LA_CHUNK) {
    dpow[threadIdx.x] = powf(decay, (float)threadIdx.x);
  }
  __syncthreads();
  const int col = lane & 15, g = lane >> 4;
  // the ten score tiles on and below the diagonal, in turn over the waves
  for (int tile = w; tile < 10; tile += 4) {
    int ti = 0, rest = tile;
    while (rest > ti) { rest -= ti + 1; ++ti; }       // tile -> (ti, sj = rest), sj <= ti
    const int sj = rest;
    floatx4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
    for (int kk = 0; kk < DP / 4; ++kk)
      acc = __builtin_amdgcn_mfma_f32_16x16x4f32(sq[(16 * ti + col) * DPS + 4 * kk + g], sk[(16 * sj + col) * DPS + 4 * kk + g],
                                                 acc, 0, 0, 0);
    const int sidx = 16 * sj + col;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int t = 16 * ti + 4 * g + r;
      float weight = 0.f;
      if (sidx <= t)
        weight = KIND == MF_LA_MEMORY ? (t < n ? expf((float)(s_decay[t] - s_decay[sidx]) + s_take[sidx]) : 0.f) : dpow[t - sidx];
      sa[t * MF_LA_VS + sidx] = acc[r] * weight;
    }
  }
  __syncthreads();
  if (KIND == MF_LA_MEMORY && blockIdx.z == 0) {
    // n_t . q_t: what n_in contributes, and the row's scores; four threads a token
    const int t = threadIdx.x >> 2, part = threadIdx.x & 3;
    float a = 0.f;
    if (t < n) {
      const float* n_in = ex.n_ws + ((size_t)c * H + h) * D;
      for (int d = part; d < D; d += 4) a = fmaf(sq[t * DPS + d], n_in[d], a);
      a *= dpow[t + 1];
      for (int s = part; s <= t; s += 4) a += sa[t * MF_LA_VS + s];
    }
    a += __shfl_xor(a, 1, MF_WAVE);
    a += __shfl_xor(a, 2, MF_WAVE);
    if (t < n && part == 0) {
      ex.den[(size_t)(t0 + t) * H + h] = a;
      ex.floor[(size_t)(t0 + t) * H + h] = ex.gates[(size_t)(t0 + t) * H + h].floor;
    }
  }
  const int cc = v0 + 16 * w + col;
  for (int ti = 0; ti < MF_LA_CHUNK / 16 && 16 * ti < n; ++ti) {
    floatx4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
    for (int kk = 0; kk < DP / 4; ++kk)
      acc = __builtin_amdgcn_mfma_f32_16x16x4f32(sq[(16 * ti + col) * DPS + 4 * kk + g], ss[(4 * kk + g) * MF_LA_VS + 16 * w + col],
                                                 acc, 0, 0, 0);
#pragma unroll
    for (int r = 0; r < 4; ++r) acc[r] *= dpow[16 * ti + 4 * g + r + 1];
#pragma unroll 4
    for (int kk = 0; kk < 4 * (ti + 1); ++kk)
      acc = __builtin_amdgcn_mfma_f32_16x16x4f32(sa[(16 * ti + col) * MF_LA_VS + 4 * kk + g], sv[(4 * kk + g) * MF_LA_VS + 16 * w + col],
                                                 acc, 0, 0, 0);
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int t = 16 * ti + 4 * g + r;
      if (t < n && cc < V) out[(size_t)(t0 + t) * H * V + h * V + cc] = acc[r];
    }
  }
}

// ------------------------------------------------------------------ norm of the heads together, and the gate
// y[t][:] = o[t][:] / sqrt(mean(o[t]^2) + eps) * w * sigmoid(gate[t][:]); gate is a column range of the
// projection row.  One workgroup per token.
template <typename OT>
__global__ __launch_bounds__(256) void gated_rmsnorm_kernel(const float* __restrict__ o, const float* __restrict__ gate,
                                                            int gate_stride, const float* __restrict__ w,
                                                            OT* __restrict__ y, int n, float eps) {
  __shared__ float scratch[4];
  const float* row = o + (size_t)blockIdx.x * n;
  const float* g = gate + (size_t)blockIdx.x * gate_stride;
  float ss = 0.f;
  for (int i = threadIdx.x; i < n; i += 256) ss = fmaf(row[i], row[i], ss);
  ss = block_sum<256>(ss, scratch);
  const float r = 1.0f / sqrtf(ss / (float)n + eps);
  for (int i = threadIdx.x; i < n; i += 256)
    y[(size_t)blockIdx.x * n + i] = from_f32<OT>(row[i] * r * w[i] * la_sigmoid(g[i]));
}

// y[t][h][:] = u / sqrt(mean(u^2) + eps) * w * act(gate[t][h][:]) with u = o[t][h][:], or, where `den` is given,
// u = o[t][h][:] / (max(|den[t][h]|, floor[t][h]) + 1e-6); w: none, one vector shared by the heads, or the heads'
// own side by side (w_stride 0 or V); act: the sigmoid or silu.  A wave per head.
template <typename OT>
__global__ __launch_bounds__(256) void gated_head_norm_kernel(const float* __restrict__ o, const float* __restrict__ den,
                                                              const float* __restrict__ floor,
                                                              const float* __restrict__ gate, int gate_stride,
                                                              const float* __restrict__ w, int w_stride,
                                                              OT* __restrict__ y, int H, int V, int silu, float eps) {
  const int t = blockIdx.x, h = blockIdx.y * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
  if (h >= H) return;
  const float* row = o + ((size_t)t * H + h) * V;
  const float* g = gate + (size_t)t * gate_stride + (size_t)h * V;
  float ss = 0.f;
  for (int i = lane; i < V; i += 64) ss = fmaf(row[i], row[i], ss);
  ss = wave_sum(ss);
  float by = 1.f;
  if (den) by = 1.0f / (fmaxf(fabsf(den[(size_t)t * H + h]), floor[(size_t)t * H + h]) + 1e-6f);
  const float r = by / sqrtf(ss * by * by / (float)V + eps);
  for (int i = lane; i < V; i += 64) {
    const float z = g[i], s = la_sigmoid(z);
    const float gain = w ? w[(size_t)h * w_stride + i] : 1.0f;
    y[((size_t)t * H + h) * V + i] = from_f32<OT>(row[i] * r * gain * (silu ? z * s : s));
  }
}

// ------------------------------------------------------------------ entry points
#define MF_LA_DISPATCH(CALL)                   \
  if (D <= 32) { CALL(8) }                     \
  else if (D <= 64) { CALL(16) }               \
  else if (D <= 128) { CALL(32) }              \
  else { CALL(64) }

MF_API int mf_la_chunk(void) { return MF_LA_CHUNK; }
MF_API int mf_memory_gate_bytes(void) { return (int)sizeof(MemoryGate); }

namespace {

template <int KIND>
int scan_sequences(const float* proj, int row_len, const int* cu_seqlens, const int* slot_ids, const float* decays,
                   float* state, float* out, int n_seqs, int H, int D, int V, const LaExtra& ex, hipStream_t stream) {
  if (n_seqs <= 0) return 0;
  if (H <= 0 || D <= 0 || V <= 0 || D > 256) return (int)hipErrorInvalidValue;
  dim3 grid(n_seqs, H, (V + 63) / 64);
#define MF_CALL(DS)                                                                                                        \
  lightning_scan_kernel<DS, KIND><<<grid, 256, 0, stream>>>(proj, row_len, cu_seqlens, slot_ids, decays, state, out, H, D, V, \
                                                            ex);
  MF_LA_DISPATCH(MF_CALL)
#undef MF_CALL
  return mf_launch_status();
}

template <int KIND>
int scan_chunks(const float* proj, int row_len, const int* chunks, int n_chunks, const int* seq_first_chunk,
                const int* slot_ids, const float* decays, float* state, float* bsum, float* out, int n_seqs, int H, int D,
                int V, const LaExtra& ex, hipStream_t stream) {
  const int* t0 = chunks;
  const int* n = chunks + n_chunks;
  dim3 grid(n_chunks, H, (V + 63) / 64);
  int rc = 0;
#define MF_CALL(DS)                                                                                                   \
  {                                                                                                                   \
    const size_t lds = sizeof(float) * (MF_LA_CHUNK * (4 * DS + 4) + MF_LA_CHUNK * MF_LA_VS);                         \
    static bool raised = false;                                                                                       \
    if (!raised && lds > 48 * 1024) {                                                                                 \
      rc = (int)hipFuncSetAttribute((const void*)lightning_chunk_sum_kernel<DS, KIND>,                                \
                                    hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);                            \
      if (rc) return rc;                                                                                              \
      raised = true;                                                                                                  \
    }                                                                                                                 \
    lightning_chunk_sum_kernel<DS, KIND><<<grid, 256, lds, stream>>>(proj, row_len, t0, n, decays, bsum, H, D, V, ex); \
  }
  MF_LA_DISPATCH(MF_CALL)
#undef MF_CALL
  rc = mf_launch_status();
  if (rc) return rc;
  const int elements = D * V + (KIND == MF_LA_MEMORY ? D : 0);
  lightning_chunk_fold_kernel<KIND><<<dim3(n_seqs, H, (elements + 255) / 256), 256, 0, stream>>>(n, seq_first_chunk, slot_ids,
                                                                                                 decays, bsum, state, H, D, V, ex);
  rc = mf_launch_status();
  if (rc) return rc;
#define MF_CALL(DS)                                                                                                   \
  {                                                                                                                   \
    const size_t lds = sizeof(float) * (2 * MF_LA_CHUNK * (4 * DS + 4) + 2 * MF_LA_CHUNK * MF_LA_VS +                 \
                                        4 * DS * MF_LA_VS + MF_LA_CHUNK + 1);                                         \
    static bool raised = false;                                                                                       \
    if (!raised && lds > 48 * 1024) {                                                                                 \
      rc = (int)hipFuncSetAttribute((const void*)lightning_chunk_out_kernel<DS, KIND>,                                \
                                    hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);                            \
      if (rc) return rc;                                                                                              \
      raised = true;                                                                                                  \
    }                                                                                                                 \
    lightning_chunk_out_kernel<DS, KIND><<<grid, 256, lds, stream>>>(proj, row_len, t0, n, decays, bsum, out, H, D, V, ex); \
  }
  MF_LA_DISPATCH(MF_CALL)
#undef MF_CALL
  return mf_launch_status();
}

}  // namespace

// proj float32 [tokens][2 H D + 2 H V]; state float32 [slots][H][D][V]; out float32 [tokens][H V]
MF_API int mf_lightning_scan(const float* proj, const int* cu_seqlens, const int* slot_ids, const float* decays,
                             float* state, float* out, int n_seqs, int H, int D, int V, hipStream_t stream) {
  return scan_sequences<MF_LA_SILU>(proj, 2 * H * D + 2 * H * V, cu_seqlens, slot_ids, decays, state, out, n_seqs, H, D, V,
                                    LaExtra{}, stream);
}

// chunks int32 [5][n_chunks]; seq_first_chunk int32 [n_seqs + 1]; bsum float32 [n_chunks][H][D][V] scratch
MF_API int mf_lightning_scan_chunked(const float* proj, const int* chunks, int n_chunks, const int* seq_first_chunk,
                                     const int* slot_ids, const float* decays, float* state, float* bsum, float* out,
                                     int n_seqs, int H, int D, int V, hipStream_t stream) {
  if (n_seqs <= 0 || n_chunks <= 0) return 0;
  if (H <= 0 || D <= 0 || V <= 0 || D > 128 || !bsum) return (int)hipErrorInvalidValue;
  return scan_chunks<MF_LA_SILU>(proj, 2 * H * D + 2 * H * V, chunks, n_chunks, seq_first_chunk, slot_ids, decays, state, bsum,
                                 out, n_seqs, H, D, V, LaExtra{}, stream);
}

// rows of row_len floats: q [H D] | k [H D] | v [H V] | ...; cos_t, sin_t [positions][rot / 2]; n_chunks 0: every
// sequence in one walk
MF_API int mf_retention_scan(float* proj, int row_len, const int* cu_seqlens, const int* chunks, int n_chunks,
                             const int* seq_first_chunk, const int* slot_ids, const float* decays, float q_scale,
                             float k_scale, const float* cos_t, const float* sin_t, int rot, const int* positions,
                             float* state, float* bsum, float* out, int n_tok, int n_seqs, int H, int D, int V,
                             hipStream_t stream) {
  if (n_tok <= 0 || n_seqs <= 0) return 0;
  if (H <= 0 || D <= 0 || V <= 0 || D > 256 || row_len < 2 * H * D + H * V || rot < 0 || rot % 2 || rot > D ||
      (rot > 0 && (!cos_t || !sin_t || !positions)))
    return (int)hipErrorInvalidValue;
  LaExtra ex{};
  ex.q_scale = q_scale;
  ex.k_scale = k_scale;
  ex.cos_t = cos_t;
  ex.sin_t = sin_t;
  ex.positions = positions;
  ex.rot = rot;
  if (n_chunks <= 0)
    return scan_sequences<MF_LA_PLAIN>(proj, row_len, cu_seqlens, slot_ids, decays, state, out, n_seqs, H, D, V, ex, stream);
  if (D > 128 || !bsum) return (int)hipErrorInvalidValue;
  if (rot > 0) {
    la_rotate_kernel<<<n_tok, 256, 0, stream>>>(proj, row_len, cos_t, sin_t, positions, 2 * H, D, rot);
    const int rc = mf_launch_status();
    if (rc) return rc;
  }
  return scan_chunks<MF_LA_PLAIN>(proj, row_len, chunks, n_chunks, seq_first_chunk, slot_ids, decays, state, bsum, out, n_seqs,
                                  H, D, V, ex, stream);
}

// rows as above, with the gates' projections in the columns off_i + h and off_f + h; state float32
// [slots][H (D V + D + column blocks)]; den, floor float32 [tokens][H]; gates [tokens][H], chunk_decay [n_chunks][H] and n_ws
// [n_chunks][H][D] scratch of the chunked form
MF_API int mf_memory_scan(const float* proj, int row_len, const int* cu_seqlens, const int* chunks, int n_chunks,
                          const int* seq_first_chunk, const int* slot_ids, float q_scale, float k_scale, int off_i, int off_f,
                          float cap, float* state, void* gates, float* chunk_decay, float* n_ws, float* bsum, float* out,
                          float* den, float* floor, int n_seqs, int H, int D, int V, hipStream_t stream) {
  if (n_seqs <= 0) return 0;
  if (H <= 0 || D <= 0 || V <= 0 || D > 256 || row_len < 2 * H * D + H * V || !den || !floor || !(cap > 0.f) || off_i < 0 ||
      off_f < 0 || off_i + H > row_len || off_f + H > row_len)
    return (int)hipErrorInvalidValue;
  LaExtra ex{};
  ex.q_scale = q_scale;
  ex.k_scale = k_scale;
  ex.off_i = off_i;
  ex.off_f = off_f;
  ex.cap = cap;
  ex.den = den;
  ex.floor = floor;
  if (n_chunks <= 0)
    return scan_sequences<MF_LA_MEMORY>(proj, row_len, cu_seqlens, slot_ids, nullptr, state, out, n_seqs, H, D, V, ex, stream);
  if (D > 128 || !bsum || !gates || !chunk_decay || !n_ws) return (int)hipErrorInvalidValue;
  ex.gates = (const MemoryGate*)gates;
  ex.chunk_decay = chunk_decay;
  ex.n_ws = n_ws;
  memory_gates_kernel<<<dim3(n_seqs, H), 64 * MF_LA_GATE_WAVES, 0, stream>>>(proj, row_len, cu_seqlens, slot_ids,
                                                                             seq_first_chunk, state, (MemoryGate*)gates,
                                                                             chunk_decay, H, D, V, off_i, off_f, cap);
  const int rc = mf_launch_status();
  if (rc) return rc;
  return scan_chunks<MF_LA_MEMORY>(proj, row_len, chunks, n_chunks, seq_first_chunk, slot_ids, nullptr, state, bsum, out, n_seqs,
                                   H, D, V, ex, stream);
}

MF_API int mf_gated_rmsnorm(const float* o, const float* gate, int gate_stride, const float* w, void* y, int y_is_bf16,
                            int rows, int n, float eps, hipStream_t stream) {
  if (rows <= 0 || n <= 0) return 0;
  if (y_is_bf16)
    gated_rmsnorm_kernel<bf16><<<rows, 256, 0, stream>>>(o, gate, gate_stride, w, (bf16*)y, n, eps);
  else
    gated_rmsnorm_kernel<float><<<rows, 256, 0, stream>>>(o, gate, gate_stride, w, (float*)y, n, eps);
  return mf_launch_status();
}

// gate: a column range of rows of gate_stride floats; w: null, [V] or [H V] (w_per_head)
MF_API int mf_gated_head_norm(const float* o, const float* den, const float* floor, const float* gate, int gate_stride,
                              const float* w, int w_per_head, void* y, int y_is_bf16, int rows, int H, int V, int silu,
                              float eps, hipStream_t stream) {
  if (rows <= 0) return 0;
  if (H <= 0 || V <= 0 || (den != nullptr) != (floor != nullptr)) return (int)hipErrorInvalidValue;
  const dim3 grid(rows, (H + 3) / 4);
  const int w_stride = w_per_head ? V : 0;
  if (y_is_bf16)
    gated_head_norm_kernel<bf16><<<grid, 256, 0, stream>>>(o, den, floor, gate, gate_stride, w, w_stride, (bf16*)y, H, V, silu, eps);
  else
    gated_head_norm_kernel<float><<<grid, 256, 0, stream>>>(o, den, floor, gate, gate_stride, w, w_stride, (float*)y, H, V, silu, eps);
  return mf_launch_status();
}
