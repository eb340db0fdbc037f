// Linear attention under a constant decay per head on the matrix cores (long bf16 portions):
//   q = silu(zq), k = silu(zk), v = silu(zv);  S_t = a S_(t-1) + k_t v_t^T;  o_t = S_t^T q_t
// (the recurrence of gated_scan.hip's KIND 3; that kernel runs decoding, short portions, fp32 and other sizes).
// A portion is cut into chunks of 64 tokens.  With i, j counting from the chunk's first token and S0 the state before it,
//   o_i = a^(i + 1) S0^T q_i + sum_(j <= i) a^(i - j) (q_i . k_j) v_j
//   S0' = a^n S0 + sum_j a^(n - 1 - j) k_j v_j^T                            (n: the chunk's tokens)
// so everything but the walk over the chunks is a product of tiles.  Three kernels:
//   decay_chunk_kernel   per (chunk, head, slice of value columns): the chunk's own sum of k v^T, fp32;
//   decay_prefix_kernel  per (sequence, head, state elements): walks the sequence's chunks from the slot's state, leaves
//                        every chunk's S0 and, at the end, the slot's new state;
//   decay_out_kernel     per (chunk, head, slice of value columns): the outputs, fp32.
// Exactness: q, k, v enter the products as bf16 (activations); the decay weights, the scores and the state are fp32 and
// enter a product as two bf16 terms (hi + lo, 16 bits of mantissa together); sums are fp32.
//
// Fragments of v_mfma_f32_16x16x32_bf16 here: lane (li = lane & 15, g = lane >> 4); operand A holds row li, operand B
// column li, at the eight k indices 4 g + j (slot j < 4) and 16 + 4 g + (j - 4) (slot j >= 4) -- the same order in both,
// which is what the transposing LDS read and the accumulator layout (row 4 g + i, column li) give without a shuffle.
#include "common.h"

namespace k8sllm {

typedef __attribute__((address_space(3))) bf16x4 ds_bf16x4;

constexpr int DSC_L = 64;          // tokens per chunk
constexpr int DSC_VS = 128;        // value columns per workgroup
constexpr int DSC_PAD = 8;         // LDS row padding, elements

struct DecayArgs {
  const bf16_t* proj;
  long ld;
  int cq, ck, cv;                  // column offsets of q, k, v
  const float* decay;              // [H]
  const int* cu_q;
  const int* seq_slots;
  const int* positions;
  int nseq, H, D, V, R;            // R heads share a group's q and k
};

__device__ __forceinline__ float fast_silu(float z) { return z * __builtin_amdgcn_rcpf(1.f + __expf(-z)); }

// 8 bf16 of a row -> silu -> 8 floats
__device__ __forceinline__ void silu8(const bf16_t* p, float* y) {
  const u32x4 u = *reinterpret_cast<const u32x4*>(p);
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    y[2 * i] = fast_silu(lo_bf(u[i]));
    y[2 * i + 1] = fast_silu(hi_bf(u[i]));
  }
}
__device__ __forceinline__ u32x4 pack8(const float* y) {
  return u32x4{pack_bf2(y[0], y[1]), pack_bf2(y[2], y[3]), pack_bf2(y[4], y[5]), pack_bf2(y[6], y[7])};
}
__device__ __forceinline__ bf16x8 join4(bf16x4 a, bf16x4 b) {
  bf16x8 r;
#pragma unroll
  for (int j = 0; j < 4; ++j) { r[j] = a[j]; r[4 + j] = b[j]; }
  return r;
}
// fragment of LDS rows read along the row: row `r`, k indices k0 + 4 g + .., k0 + 16 + 4 g + ..
__device__ __forceinline__ bf16x8 row_frag(const bf16_t* base, int stride, int r, int k0, int g) {
  const bf16_t* p = base + r * stride + k0 + 4 * g;
  return join4(*reinterpret_cast<const bf16x4*>(p), *reinterpret_cast<const bf16x4*>(p + 16));
}
// fragment across LDS rows: column c0 + li, k indices are the rows k0 + 4 g + .., k0 + 16 + 4 g + ..
__device__ __forceinline__ bf16x8 col_frag(bf16_t* base, int stride, int c0, int k0, int li, int g) {
  bf16_t* p = base + (k0 + 4 * g + (li >> 2)) * stride + c0 + 4 * (li & 3);
  return join4(__builtin_amdgcn_ds_read_tr16_b64_v4bf16((ds_bf16x4*)p),
               __builtin_amdgcn_ds_read_tr16_b64_v4bf16((ds_bf16x4*)(p + 16 * stride)));
}
// value columns [v0, v0 + 16 NT) of the chunk's tokens into LDS (silu, bf16); tokens and columns outside are zero
__device__ __forceinline__ void stage_v(bf16_t* vl, int stride, const DecayArgs& A, int hd, int a0, int n, int v0, int cols) {
  const int cpr = cols / 8;
  for (int idx = threadIdx.x; idx < DSC_L * cpr; idx += blockDim.x) {
    const int r = idx / cpr, c = (idx - r * cpr) * 8;
    u32x4 w = u32x4{0u, 0u, 0u, 0u};
    if (r < n && v0 + c < A.V) {
      float y[8];
      silu8(A.proj + (size_t)(a0 + r) * A.ld + A.cv + (size_t)hd * A.V + v0 + c, y);
      w = pack8(y);
    }
    *reinterpret_cast<u32x4*>(vl + r * stride + c) = w;
  }
}

// A chunk / state record: tile (nt, dt) of 16 key channels x 16 value columns in accumulator order, element
// ((nt DT + dt) 64 + lane) 4 + i = S[16 dt + 4 g + i][16 nt + li], DT = 2 KK tiles of key channels (zero-padded).
template <int KK, int NTW>
__global__ __launch_bounds__(256) void decay_chunk_kernel(float* __restrict__ loc, DecayArgs A) {
  constexpr int DT = 2 * KK, DP = 32 * KK, LDK = DP + DSC_PAD;
  extern __shared__ __attribute__((aligned(16))) char smem_d[];
  const WkvChunk ck = wkv_find_chunk(blockIdx.x, A.cu_q, A.positions, A.nseq, DSC_L);
  if (ck.s < 0) return;
  const int hd = blockIdx.y, v0 = blockIdx.z * DSC_VS;
  const int a0 = A.cu_q[ck.s] + ck.c * DSC_L, n = min(DSC_L, A.cu_q[ck.s + 1] - a0);
  const int NT = (min(DSC_VS, A.V - v0) + 15) / 16, LDV = 16 * NT + DSC_PAD;
  bf16_t* khi = reinterpret_cast<bf16_t*>(smem_d);       // [64][LDK]
  bf16_t* klo = khi + DSC_L * LDK;
  bf16_t* vl = klo + DSC_L * LDK;                        // [64][LDV]
  const float dec = A.decay[hd];
  for (int idx = threadIdx.x; idx < DSC_L * (DP / 8); idx += blockDim.x) {
    const int r = idx / (DP / 8), c = (idx - r * (DP / 8)) * 8;
    u32x4 hi = u32x4{0u, 0u, 0u, 0u}, lo = hi;
    if (r < n && c < A.D) {
      float y[8], h8[8], l8[8];
      silu8(A.proj + (size_t)(a0 + r) * A.ld + A.ck + (size_t)(hd / A.R) * A.D + c, y);
      const float w = powf(dec, (float)(n - 1 - r));
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        const float f = bf_round(y[i]) * w;
        h8[i] = bf_round(f);
        l8[i] = f - h8[i];
      }
      hi = pack8(h8);
      lo = pack8(l8);
    }
    *reinterpret_cast<u32x4*>(khi + r * LDK + c) = hi;
    *reinterpret_cast<u32x4*>(klo + r * LDK + c) = lo;
  }
  stage_v(vl, LDV, A, hd, a0, n, v0, 16 * NT);
  __syncthreads();
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, li = lane & 15, g = lane >> 4;
  const int ntt = (A.V + 15) / 16;
  f32x4 acc[NTW][DT];
#pragma unroll
  for (int x = 0; x < NTW; ++x)
#pragma unroll
    for (int d = 0; d < DT; ++d) acc[x][d] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int k0 = 0; k0 < DSC_L; k0 += 32) {
    if (k0 >= n) break;
    bf16x8 vf[NTW];
#pragma unroll
    for (int x = 0; x < NTW; ++x) {
      const int nt = wave * NTW + x;
      vf[x] = col_frag(vl, LDV, 16 * (nt < NT ? nt : 0), k0, li, g);
    }
#pragma unroll
    for (int d = 0; d < DT; ++d) {
      const bf16x8 ah = col_frag(khi, LDK, 16 * d, k0, li, g), al = col_frag(klo, LDK, 16 * d, k0, li, g);
#pragma unroll
      for (int x = 0; x < NTW; ++x) {
        acc[x][d] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(al, vf[x], acc[x][d], 0, 0, 0);
        acc[x][d] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ah, vf[x], acc[x][d], 0, 0, 0);
      }
    }
  }
  float* rec = loc + ((size_t)blockIdx.x * A.H + hd) * ((size_t)ntt * DT * 256);
#pragma unroll
  for (int x = 0; x < NTW; ++x) {
    const int nt = wave * NTW + x;
    if (nt >= NT) continue;
#pragma unroll
    for (int d = 0; d < DT; ++d)
      *reinterpret_cast<f32x4*>(rec + (((size_t)(v0 / 16 + nt) * DT + d) * 64 + lane) * 4) = acc[x][d];
  }
}

// Thread: the four elements of one lane of one tile.  start (bf16 hi, then lo, per chunk): the B fragments of the state
// before the chunk, ((nt KK + kk) 64 + lane) 8 + slot.
__global__ __launch_bounds__(256) void decay_prefix_kernel(bf16_t* __restrict__ start, const float* __restrict__ loc,
                                                           float* __restrict__ state, DecayArgs A, int KK) {
  const int s = blockIdx.x, hd = blockIdx.y;
  int first = 0;
  for (int y = 0; y < s; ++y) {
    const int a = A.cu_q[y], len = A.cu_q[y + 1] - a;
    first += (len > 0 && A.positions[a] >= 0) ? (len + DSC_L - 1) / DSC_L : 0;
  }
  const int a = A.cu_q[s], len = A.cu_q[s + 1] - a;
  if (len <= 0 || A.positions[a] < 0) return;
  const int nch = (len + DSC_L - 1) / DSC_L;
  const int DT = 2 * KK, ntt = (A.V + 15) / 16, nvec = ntt * DT * 64;
  const int e = blockIdx.z * blockDim.x + threadIdx.x;
  if (e >= nvec) return;
  const int lane = e & 63, tile = e >> 6, nt = tile / DT, dt = tile - nt * DT;
  const int v = 16 * nt + (lane & 15), d0 = 16 * dt + 4 * (lane >> 4);
  const size_t recf = (size_t)nvec * 4;                  // floats of a chunk's record
  float* st = state + ((size_t)A.seq_slots[s] * A.H + hd) * ((size_t)A.D * A.V);
  const float dec = A.decay[hd], full = powf(dec, (float)DSC_L);
  const bool zero = A.positions[a] == 0;
  float X[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) X[i] = (!zero && d0 + i < A.D && v < A.V) ? st[(size_t)(d0 + i) * A.V + v] : 0.f;
  const size_t sofs = (((size_t)nt * KK + (dt >> 1)) * 64 + lane) * 8 + (dt & 1) * 4;
  const float* lp = loc + ((size_t)first * A.H + hd) * recf + (size_t)e * 4;
  const size_t lstep = (size_t)A.H * recf;
  constexpr int PF = 8;                                  // records in flight
  f32x4 buf[PF];
#pragma unroll
  for (int i = 0; i < PF; ++i)
    if (i < nch) buf[i] = *reinterpret_cast<const f32x4*>(lp + i * lstep);
  for (int c0 = 0; c0 < nch; c0 += PF) {
#pragma unroll
    for (int i = 0; i < PF; ++i) {
      const int c = c0 + i;
      if (c < nch) {
        const f32x4 U = buf[i];
        if (c + PF < nch) buf[i] = *reinterpret_cast<const f32x4*>(lp + (c + PF) * lstep);
        if (c > 0 || !zero) {
          float h[4], l[4];
#pragma unroll
          for (int j = 0; j < 4; ++j) {
            h[j] = bf_round(X[j]);
            l[j] = X[j] - h[j];
          }
          bf16_t* sp = start + ((size_t)(first + c) * A.H + hd) * (2 * recf) + sofs;
          *reinterpret_cast<uint2*>(sp) = make_uint2(pack_bf2(h[0], h[1]), pack_bf2(h[2], h[3]));
          *reinterpret_cast<uint2*>(sp + recf) = make_uint2(pack_bf2(l[0], l[1]), pack_bf2(l[2], l[3]));
        }
        const float w = c + 1 < nch ? full : powf(dec, (float)(len - c * DSC_L));
#pragma unroll
        for (int j = 0; j < 4; ++j) X[j] = fmaf(w, X[j], U[j]);
      }
    }
  }
#pragma unroll
  for (int i = 0; i < 4; ++i)
    if (d0 + i < A.D && v < A.V) st[(size_t)(d0 + i) * A.V + v] = X[i];
}

// Waves: first each the scores of its 16 queries against the keys up to them, weighted, into LDS; then each its value
// columns for all 64 queries.
template <int KK, int NTW>
__global__ __launch_bounds__(256) void decay_out_kernel(float* __restrict__ out, const bf16_t* __restrict__ start,
                                                        DecayArgs A) {
  constexpr int DT = 2 * KK, DP = 32 * KK, LDK = DP + DSC_PAD, LDP = DSC_L + DSC_PAD;
  extern __shared__ __attribute__((aligned(16))) char smem_d[];
  __shared__ float pw[DSC_L + 1];
  const WkvChunk ck = wkv_find_chunk(blockIdx.x, A.cu_q, A.positions, A.nseq, DSC_L);
  if (ck.s < 0) return;
  const int hd = blockIdx.y, v0 = blockIdx.z * DSC_VS;
  const int a0 = A.cu_q[ck.s] + ck.c * DSC_L, n = min(DSC_L, A.cu_q[ck.s + 1] - a0);
  const bool zero = A.positions[a0] == 0;
  const int NT = (min(DSC_VS, A.V - v0) + 15) / 16, LDV = 16 * NT + DSC_PAD;
  bf16_t* kq = reinterpret_cast<bf16_t*>(smem_d);        // [64][LDK]: keys, then queries
  bf16_t* ph = kq + DSC_L * LDK;                         // [64][LDP]
  bf16_t* pl = ph + DSC_L * LDP;
  bf16_t* vl = pl + DSC_L * LDP;                         // [64][LDV]
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, li = lane & 15, g = lane >> 4;
  if (threadIdx.x <= DSC_L) pw[threadIdx.x] = powf(A.decay[hd], (float)threadIdx.x);
  for (int idx = threadIdx.x; idx < DSC_L * (DP / 8); idx += blockDim.x) {
    const int r = idx / (DP / 8), c = (idx - r * (DP / 8)) * 8;
    u32x4 w = u32x4{0u, 0u, 0u, 0u};
    if (r < n && c < A.D) {
      float y[8];
      silu8(A.proj + (size_t)(a0 + r) * A.ld + A.ck + (size_t)(hd / A.R) * A.D + c, y);
      w = pack8(y);
    }
    *reinterpret_cast<u32x4*>(kq + r * LDK + c) = w;
  }
  stage_v(vl, LDV, A, hd, a0, n, v0, 16 * NT);
  // this wave's queries: row 16 wave + li, channels in fragment order
  bf16x8 qf[KK];
  {
    const int r = 16 * wave + li;
    const bf16_t* qp = A.proj + (size_t)(a0 + r) * A.ld + A.cq + (size_t)(hd / A.R) * A.D;
#pragma unroll
    for (int kk = 0; kk < KK; ++kk)
#pragma unroll
      for (int hf = 0; hf < 2; ++hf) {
        const int d = 32 * kk + 16 * hf + 4 * g;
        uint2 u = make_uint2(0u, 0u);
        if (r < n && d < A.D) u = *reinterpret_cast<const uint2*>(qp + d);
        const float f[4] = {lo_bf(u.x), hi_bf(u.x), lo_bf(u.y), hi_bf(u.y)};
#pragma unroll
        for (int j = 0; j < 4; ++j) qf[kk][4 * hf + j] = (__bf16)fast_silu(f[j]);
      }
  }
  __syncthreads();
  const bool active = 16 * wave < n;
  if (active) {
#pragma unroll
    for (int jt = 0; jt < 4; ++jt) {
      if (jt > (wave | 1)) break;
      f32x4 sc = f32x4{0.f, 0.f, 0.f, 0.f};
      if (jt <= wave) {
#pragma unroll
        for (int kk = 0; kk < KK; ++kk)
          sc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(row_frag(kq, LDK, 16 * jt + li, 32 * kk, g), qf[kk], sc, 0, 0, 0);
      }
      // sc[i]: key 16 jt + 4 g + i, query 16 wave + li
      float h[4], l[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int age = 16 * wave + li - (16 * jt + 4 * g + i);
        const float p = age >= 0 ? sc[i] * pw[age] : 0.f;
        h[i] = bf_round(p);
        l[i] = p - h[i];
      }
      const int o = (16 * wave + li) * LDP + 16 * jt + 4 * g;
      *reinterpret_cast<uint2*>(ph + o) = make_uint2(pack_bf2(h[0], h[1]), pack_bf2(h[2], h[3]));
      *reinterpret_cast<uint2*>(pl + o) = make_uint2(pack_bf2(l[0], l[1]), pack_bf2(l[2], l[3]));
    }
  }
  __syncthreads();
#pragma unroll
  for (int kk = 0; kk < KK; ++kk) {   // the queries take the keys' place
    bf16_t* p = kq + (16 * wave + li) * LDK + 32 * kk + 4 * g;
    bf16x4 x, y;
#pragma unroll
    for (int j = 0; j < 4; ++j) { x[j] = qf[kk][j]; y[j] = qf[kk][4 + j]; }
    *reinterpret_cast<bf16x4*>(p) = x;
    *reinterpret_cast<bf16x4*>(p + 16) = y;
  }
  __syncthreads();
  f32x4 acc[NTW][4];
#pragma unroll
  for (int x = 0; x < NTW; ++x)
#pragma unroll
    for (int rt = 0; rt < 4; ++rt) acc[x][rt] = f32x4{0.f, 0.f, 0.f, 0.f};
  const int ntt = (A.V + 15) / 16;
  if (!zero) {
    const size_t recf = (size_t)ntt * DT * 256;
    const bf16_t* sp = start + ((size_t)blockIdx.x * A.H + hd) * (2 * recf);
#pragma unroll
    for (int kk = 0; kk < KK; ++kk) {
      bf16x8 sh[NTW], sl[NTW];
#pragma unroll
      for (int x = 0; x < NTW; ++x) {
        const int nt = wave * NTW + x;
        const size_t o = (((size_t)(v0 / 16 + (nt < NT ? nt : 0)) * KK + kk) * 64 + lane) * 8;
        sh[x] = *reinterpret_cast<const bf16x8*>(sp + o);
        sl[x] = *reinterpret_cast<const bf16x8*>(sp + recf + o);
      }
#pragma unroll
      for (int rt = 0; rt < 4; ++rt) {
        const bf16x8 a = row_frag(kq, LDK, 16 * rt + li, 32 * kk, g);
#pragma unroll
        for (int x = 0; x < NTW; ++x) {
          acc[x][rt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, sl[x], acc[x][rt], 0, 0, 0);
          acc[x][rt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, sh[x], acc[x][rt], 0, 0, 0);
        }
      }
    }
#pragma unroll
    for (int rt = 0; rt < 4; ++rt)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const float w = pw[16 * rt + 4 * g + i + 1];
#pragma unroll
        for (int x = 0; x < NTW; ++x) acc[x][rt][i] *= w;
      }
  }
#pragma unroll
  for (int k0 = 0; k0 < DSC_L; k0 += 32) {
    if (k0 >= n) break;
    bf16x8 vf[NTW];
#pragma unroll
    for (int x = 0; x < NTW; ++x) {
      const int nt = wave * NTW + x;
      vf[x] = col_frag(vl, LDV, 16 * (nt < NT ? nt : 0), k0, li, g);
    }
#pragma unroll
    for (int rt = k0 / 16; rt < 4; ++rt) {
      if (16 * rt >= n) break;                           // those rows' scores were not written
      const bf16x8 a1 = row_frag(pl, LDP, 16 * rt + li, k0, g), a0f = row_frag(ph, LDP, 16 * rt + li, k0, g);
#pragma unroll
      for (int x = 0; x < NTW; ++x) {
        acc[x][rt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a1, vf[x], acc[x][rt], 0, 0, 0);
        acc[x][rt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a0f, vf[x], acc[x][rt], 0, 0, 0);
      }
    }
  }
#pragma unroll
  for (int x = 0; x < NTW; ++x) {
    const int nt = wave * NTW + x, col = v0 + 16 * nt + li;
    if (nt >= NT || col >= A.V) continue;
#pragma unroll
    for (int rt = 0; rt < 4; ++rt)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int r = 16 * rt + 4 * g + i;
        if (r < n) out[(size_t)(a0 + r) * A.H * A.V + (size_t)hd * A.V + col] = acc[x][rt][i];
      }
  }
}

}  // namespace k8sllm

using namespace k8sllm;

// Whether these sizes run here (else k8s_gated_scan): rows of 16 bytes, at most 128 key channels.
extern "C" int k8s_decay_scan_ok(int D, int V) { return D > 0 && D <= 128 && D % 8 == 0 && V > 0 && V <= 256 && V % 8 == 0; }

// Bytes of workspace: per chunk and head one fp32 record and one record of two bf16 terms.
extern "C" long long k8s_decay_scan_workspace(int T, int nseq, int H, int D, int V) {
  const long long chunks = (T + DSC_L - 1) / DSC_L + nseq;
  const long long rec = (long long)((V + 15) / 16) * 2 * ((D + 31) / 32) * 256;
  return chunks * H * rec * 8;
}

// proj bf16 [T, ld] (16-byte aligned rows and parts); out fp32 [T, H V]; state [slots, H, D V] fp32, updated in place.
extern "C" int k8s_decay_scan(float* out, const void* proj, long ld, int cq, int ck, int cv, const float* decay,
                              float* state, const int* cu_q, const int* seq_slots, const int* positions, int nseq, int H,
                              int D, int V, int R, int T, void* ws, hipStream_t s) {
  if (T <= 0 || nseq <= 0) return 0;
  if (!k8s_decay_scan_ok(D, V) || H <= 0 || H > 65535 || R <= 0 || H % R || ws == nullptr || decay == nullptr) return -1;
  if (ld % 8 || cq % 8 || ck % 8 || cv % 8 || ((uintptr_t)proj & 15)) return -1;
  const DecayArgs A{(const bf16_t*)proj, ld, cq, ck, cv, decay, cu_q, seq_slots, positions, nseq, H, D, V, R};
  const int chunks = (T + DSC_L - 1) / DSC_L + nseq, KK = (D + 31) / 32;
  const int slices = (V + DSC_VS - 1) / DSC_VS, ntt = (V + 15) / 16;
  const size_t recf = (size_t)ntt * 2 * KK * 256;
  float* loc = (float*)ws;
  bf16_t* start = (bf16_t*)(loc + (size_t)chunks * H * recf);
  const int nt = ntt < 8 ? ntt : 8, LDK = 32 * KK + DSC_PAD, LDV = 16 * nt + DSC_PAD;
  const size_t lds1 = (size_t)DSC_L * (2 * LDK + LDV) * 2;
  const size_t lds3 = (size_t)DSC_L * (LDK + 2 * (DSC_L + DSC_PAD) + LDV) * 2;
  const dim3 grid(chunks, H, slices), pgrid(nseq, H, (unsigned)((recf / 4 + 255) / 256));
#define K8S_DS(KK_, NTW)                                                              \
  do {                                                                                \
    decay_chunk_kernel<KK_, NTW><<<grid, 256, lds1, s>>>(loc, A);                     \
    decay_prefix_kernel<<<pgrid, 256, 0, s>>>(start, loc, state, A, KK);              \
    decay_out_kernel<KK_, NTW><<<grid, 256, lds3, s>>>(out, start, A);                \
  } while (0)
#define K8S_DS_N(KK_)                 \
  do {                                \
    if (nt <= 4) K8S_DS(KK_, 1);      \
    else K8S_DS(KK_, 2);              \
  } while (0)
  if (KK == 1) K8S_DS_N(1);
  else if (KK == 2) K8S_DS_N(2);
  else if (KK == 3) K8S_DS_N(3);
  else K8S_DS_N(4);
#undef K8S_DS_N
#undef K8S_DS
  return (int)hipGetLastError();
}
