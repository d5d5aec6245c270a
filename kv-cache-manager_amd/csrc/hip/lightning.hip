// A matrix state per head with a constant decay, for runs of rows, in matrix form (gated_state.hip walks the same recurrence row
// by row: steps of single rows and short runs).  S_t = decay S_(t-1) + k_t v_t^T, o_t = S_t^T q_t, with q, k and v silu of what
// is given where asked for.  A chunk of up to 64 rows that starts from the state S gives
//
//   o_i = decay^(i+1) S^T q_i + sum over j <= i of decay^(i-j) (q_i . k_j) v_j
//   S  <- decay^n S + sum over j of decay^(n-1-j) k_j v_j^T                      (n rows in the chunk)
//
// which are four products: Q S, Q K^T, (its masked and decayed result) V and K^T V, all in 32-bit on the matrix cores
// (v_mfma_f32_16x16x4_f32: inputs, products and sums are 32-bit, nothing is rounded to 16).  The powers of every head's decay
// come as a table, made in double precision.
//
// Runs of more than `piece` rows are walked in pieces, all pieces at once: every piece's own part of the state (the K^T V
// products alone), then the states that enter the pieces, one after another (S <- decay^piece S + part, element by element),
// then every piece again from the state that enters it, now with outputs.  Runs of at most a piece are one launch.
//
// A workgroup of four waves (or eight: CS 2, two waves share a row tile and halve its columns) takes one (sequence, piece, head)
// and a stretch of DVT value columns.  K and V of a chunk are staged through LDS (the next chunk's on their way in registers
// meanwhile), a wave holds its 16 rows of q in registers and computes their outputs; the state stays in accumulators, a quarter of
// the key dimension a wave, and passes through LDS once per chunk.
// The sum over k of a 16 x 16 x 4 instruction may take k in any order: a lane group g takes the four consecutive k = 4 g .. 4 g + 3
// of every sixteen over four instructions, so that what lies along k is read 16 bytes at a time.
#include "common.h"
#include "kvcm_hip.h"

namespace kvcm {

typedef __attribute__((__vector_size__(4 * sizeof(float)))) float f32x4;

constexpr int kLtRows = 64;      // rows of a chunk

struct LightningArgs {
  const float *q, *k, *v;      // 32-bit rows
  int ldq, ldk, ldv;
  const float* powers;         // [heads][kLtRows + 2]: decay^0 .. decay^64, decay^piece
  float* o;
  int ldo;
  float* state;                // [slots, heads, dk, dv]
  const int *run_start, *seq_start, *state_slots;
  int heads, dk, dv, col_blocks, silu_in;
  float* carry;                // pieces: per (piece, head) [dk][dv]
  int piece, pieces_per_seq;   // piece 0: one piece a run
};

// where a piece's part of the carry lies (pieces of all sequences are numbered so that no two meet)
__device__ __forceinline__ int lightning_place(int run0, int s, int p, int piece) { return run0 / piece + s + p; }

// four values of a row of n from place i on; zero where the row is none of the run's (``in``) or ends.  Loads are unconditional,
// from places clamped into the row, and masked afterwards (a branch around a load would make each wait for the one before).
template <bool WIDE>
__device__ __forceinline__ float4 load4(const float* row, int i, int n, bool in) {
  if constexpr (WIDE) {      // (n and i are multiples of four)
    const float4 x = *reinterpret_cast<const float4*>(row + (i < n ? i : 0));
    return in && i < n ? x : float4{0.f, 0.f, 0.f, 0.f};
  }
  float x[4];
#pragma unroll
  for (int e = 0; e < 4; ++e) {
    const float y = row[i + e < n ? i + e : 0];
    x[e] = in && i + e < n ? y : 0.f;
  }
  return float4{x[0], x[1], x[2], x[3]};
}

// (by the hardware's exp2 and reciprocal, about one unit of the last place each: the exact functions cost as much as the products)
__device__ __forceinline__ float4 silu4(float4 x) { return float4{silu<bf16_t>(x.x), silu<bf16_t>(x.y), silu<bf16_t>(x.z), silu<bf16_t>(x.w)}; }

// PARTS: the first of the three launches (no outputs; the piece's own part of the state goes to the carry)
template <int DKP, int DVT, int CS, bool WIDE, bool PARTS>
__global__ void __launch_bounds__(256 * CS) lightning_kernel(LightningArgs A) {
  constexpr int C = kLtRows, KP = DKP + 4, VP = DVT + 4, PP = C + 4;      // pitches: rows four apart lie 16 banks apart
  constexpr int BT = DKP / 64, CT = DVT / 16 / CS, KS = DKP / 16, NT = 256 * CS;
  __shared__ __attribute__((aligned(16))) float Ks[C][KP];
  __shared__ __attribute__((aligned(16))) float Vs[C][VP];
  __shared__ __attribute__((aligned(16))) float Ss[PARTS ? 1 : DKP][VP];
  __shared__ __attribute__((aligned(16))) float Ps[PARTS ? 1 : 4][16][PP];
  __shared__ float pw[C + 1];
  const int head = blockIdx.x / A.col_blocks, c0 = (blockIdx.x % A.col_blocks) * DVT;
  const int s = blockIdx.y / A.pieces_per_seq, p = blockIdx.y % A.pieces_per_seq;
  const int tid = threadIdx.x, wave = (tid / kWave) % 4, half = tid / 256, lane = tid % kWave, col = lane % 16, g = lane / 16;
  const int cw = half * CT * 16;      // where this wave's columns of the stretch start
  const int dk = A.dk, dv = A.dv;
  const int run0 = A.run_start[s], run1 = A.run_start[s + 1], slot = A.state_slots[s];
  const bool pieces = A.piece > 0;
  const int r0 = pieces ? run0 + p * A.piece : run0;
  const int r1 = pieces && run1 - r0 > A.piece ? r0 + A.piece : run1;
  if (r1 <= r0) return;
  const bool last = r1 == run1;
  if (PARTS && (last || slot < 0)) return;      // nothing follows the last piece
  const int cols = dv - c0 < DVT ? dv - c0 : DVT;
  if (slot < 0) {
    for (int e = tid; e < (r1 - r0) * cols; e += NT) A.o[size_t(r0 + e / cols) * A.ldo + size_t(head) * dv + c0 + e % cols] = 0.f;
    return;
  }
  if (tid <= C) pw[tid] = A.powers[size_t(head) * (C + 2) + tid];
  float* part = pieces ? A.carry + (size_t(lightning_place(run0, s, p, A.piece)) * A.heads + head) * dk * dv : nullptr;
  float* home = A.state + (size_t(slot) * A.heads + head) * dk * dv;

  // this wave's quarter of the state: row tiles of 16 keys by column tiles of 16 values; a lane holds rows 4 g + i of column col
  f32x4 S[BT][CT];
  {
    const float* src = PARTS ? nullptr : pieces ? part : A.seq_start[s] == 0 ? nullptr : home;
#pragma unroll
    for (int b = 0; b < BT; ++b)
#pragma unroll
      for (int ct = 0; ct < CT; ++ct)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int key = (wave * BT + b) * 16 + g * 4 + i, c = cw + ct * 16 + col;
          S[b][ct][i] = src && key < dk && c < cols ? src[size_t(key) * dv + c0 + c] : 0.f;
        }
  }

  constexpr int KQ = C * DKP / 4 / NT, VQ = C * DVT / 4 / NT;
  float4 kreg[KQ], vreg[VQ], qreg[PARTS ? 1 : KS];
  auto request = [&](int t0) {      // rows t0 .. t0 + 63 of the piece; what lies outside is zero
#pragma unroll
    for (int n = 0; n < KQ; ++n) {
      const int e = tid + n * NT, row = e / (DKP / 4), i = (e % (DKP / 4)) * 4;
      kreg[n] = load4<WIDE>(A.k + size_t(t0 + row < r1 ? t0 + row : r1 - 1) * A.ldk + size_t(head) * dk, i, dk, t0 + row < r1);
    }
#pragma unroll
    for (int n = 0; n < VQ; ++n) {
      const int e = tid + n * NT, row = e / (DVT / 4), c = (e % (DVT / 4)) * 4;
      vreg[n] = load4<WIDE>(A.v + size_t(t0 + row < r1 ? t0 + row : r1 - 1) * A.ldv + size_t(head) * dv + c0, c, cols, t0 + row < r1);
    }
    if constexpr (!PARTS) {
      const int row = t0 + wave * 16 + col;
      const float* qrow = A.q + size_t(row < r1 ? row : r1 - 1) * A.ldq + size_t(head) * dk;
#pragma unroll
      for (int ks = 0; ks < KS; ++ks) qreg[ks] = load4<WIDE>(qrow, ks * 16 + g * 4, dk, row < r1);
    }
  };

  request(r0);
  for (int t0 = r0; t0 < r1; t0 += C) {
    const int n = r1 - t0 < C ? r1 - t0 : C;
    __syncthreads();      // the chunk before is done with Ks, Vs and Ss
#pragma unroll
    for (int m = 0; m < KQ; ++m) {
      const int e = tid + m * NT;
      *reinterpret_cast<float4*>(&Ks[e / (DKP / 4)][(e % (DKP / 4)) * 4]) = A.silu_in ? silu4(kreg[m]) : kreg[m];
    }
#pragma unroll
    for (int m = 0; m < VQ; ++m) {
      const int e = tid + m * NT;
      *reinterpret_cast<float4*>(&Vs[e / (DVT / 4)][(e % (DVT / 4)) * 4]) = A.silu_in ? silu4(vreg[m]) : vreg[m];
    }
    float4 qf[PARTS ? 1 : KS];
    if constexpr (!PARTS) {
#pragma unroll
      for (int ks = 0; ks < KS; ++ks) qf[ks] = A.silu_in ? silu4(qreg[ks]) : qreg[ks];
#pragma unroll
      for (int b = 0; b < BT; ++b)
#pragma unroll
        for (int ct = 0; ct < CT; ++ct)
#pragma unroll
          for (int i = 0; i < 4; ++i) Ss[(wave * BT + b) * 16 + g * 4 + i][cw + ct * 16 + col] = S[b][ct][i];
    }
    __syncthreads();
    if (t0 + C < r1) request(t0 + C);      // on its way while this chunk is multiplied

    if constexpr (!PARTS) {
      const bool busy = wave * 16 < n;
      if (busy) {
        // Q K^T of this wave's rows with the rows up to its own, masked and decayed, to LDS as the next product's first operand
#pragma unroll
        for (int jt = 0; jt < 4; ++jt) {
          if (jt > wave) break;
          if (CS > 1 && jt % CS != half) continue;      // (the row tile's other wave makes these)
          f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
          for (int ks = 0; ks < KS; ++ks) {
            const float4 kf = *reinterpret_cast<const float4*>(&Ks[jt * 16 + col][ks * 16 + g * 4]);
            acc = __builtin_amdgcn_mfma_f32_16x16x4f32(qf[ks].x, kf.x, acc, 0, 0, 0);
            acc = __builtin_amdgcn_mfma_f32_16x16x4f32(qf[ks].y, kf.y, acc, 0, 0, 0);
            acc = __builtin_amdgcn_mfma_f32_16x16x4f32(qf[ks].z, kf.z, acc, 0, 0, 0);
            acc = __builtin_amdgcn_mfma_f32_16x16x4f32(qf[ks].w, kf.w, acc, 0, 0, 0);
          }
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            const int back = (wave - jt) * 16 + g * 4 + i - col;      // row - column
            Ps[wave][g * 4 + i][jt * 16 + col] = back >= 0 ? acc[i] * pw[back] : 0.f;
          }
        }
        __builtin_amdgcn_wave_barrier();
      }
      if constexpr (CS > 1) __syncthreads();
      if (busy) {
        f32x4 acc[CT];
#pragma unroll
        for (int ct = 0; ct < CT; ++ct) acc[ct] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int ks = 0; ks < KS; ++ks) {
          const float qe[4] = {qf[ks].x, qf[ks].y, qf[ks].z, qf[ks].w};
#pragma unroll
          for (int e = 0; e < 4; ++e)
#pragma unroll
            for (int ct = 0; ct < CT; ++ct)
              acc[ct] = __builtin_amdgcn_mfma_f32_16x16x4f32(qe[e], Ss[ks * 16 + g * 4 + e][cw + ct * 16 + col], acc[ct], 0, 0, 0);
        }
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const float f = pw[wave * 16 + g * 4 + i + 1];
#pragma unroll
          for (int ct = 0; ct < CT; ++ct) acc[ct][i] *= f;
        }
#pragma unroll
        for (int jt = 0; jt < 4; ++jt) {
          if (jt > wave) break;
          const float4 pf = *reinterpret_cast<const float4*>(&Ps[wave][col][jt * 16 + g * 4]);
          const float pe[4] = {pf.x, pf.y, pf.z, pf.w};
#pragma unroll
          for (int e = 0; e < 4; ++e)
#pragma unroll
            for (int ct = 0; ct < CT; ++ct)
              acc[ct] = __builtin_amdgcn_mfma_f32_16x16x4f32(pe[e], Vs[jt * 16 + g * 4 + e][cw + ct * 16 + col], acc[ct], 0, 0, 0);
        }
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int row = wave * 16 + g * 4 + i;
          if (row >= n) continue;
          float* dst = A.o + size_t(t0 + row) * A.ldo + size_t(head) * dv + c0;
#pragma unroll
          for (int ct = 0; ct < CT; ++ct)
            if (cw + ct * 16 + col < cols) dst[cw + ct * 16 + col] = acc[ct][i];
        }
      }
      if (t0 + C >= r1 && !last) break;      // the state that leaves this piece is another piece's business
    }
    const float keep = pw[n];
#pragma unroll
    for (int b = 0; b < BT; ++b)
#pragma unroll
      for (int ct = 0; ct < CT; ++ct)
#pragma unroll
        for (int i = 0; i < 4; ++i) S[b][ct][i] *= keep;
    const int tiles = (n + 15) / 16;
    for (int jt = 0; jt < tiles; ++jt)
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int j = jt * 16 + g * 4 + e, left = n - 1 - j;      // (rows beyond the chunk's are zero)
        const float w = pw[left > 0 ? left : 0];
        float kf[BT];
#pragma unroll
        for (int b = 0; b < BT; ++b) kf[b] = Ks[j][(wave * BT + b) * 16 + col] * w;
#pragma unroll
        for (int ct = 0; ct < CT; ++ct) {
          const float vf = Vs[j][cw + ct * 16 + col];
#pragma unroll
          for (int b = 0; b < BT; ++b) S[b][ct] = __builtin_amdgcn_mfma_f32_16x16x4f32(kf[b], vf, S[b][ct], 0, 0, 0);
        }
      }
  }
  if (PARTS || last) {
    float* dst = PARTS ? part : home;
#pragma unroll
    for (int b = 0; b < BT; ++b)
#pragma unroll
      for (int ct = 0; ct < CT; ++ct)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int key = (wave * BT + b) * 16 + g * 4 + i, c = cw + ct * 16 + col;
          if (key < dk && c < cols) dst[size_t(key) * dv + c0 + c] = S[b][ct][i];
        }
  }
}

// the states that enter a run's pieces, from its slot (or zero): carry[piece] <- S, then S <- decay^piece S + what the piece had
// left there.  grid (element blocks, heads, sequences); an element's chain is one thread's.
__global__ void __launch_bounds__(256) lightning_pass_kernel(LightningArgs A) {
  const int e = blockIdx.x * 256 + threadIdx.x, head = blockIdx.y, s = blockIdx.z;
  const int run0 = A.run_start[s], len = A.run_start[s + 1] - run0, slot = A.state_slots[s], size = A.dk * A.dv;
  if (len <= 0 || slot < 0 || e >= size) return;
  const int n = (len + A.piece - 1) / A.piece;
  const float keep = A.powers[size_t(head) * (kLtRows + 2) + kLtRows + 1];
  float cur = A.seq_start[s] == 0 ? 0.f : A.state[(size_t(slot) * A.heads + head) * size + e];
  float* at = A.carry + (size_t(lightning_place(run0, s, 0, A.piece)) * A.heads + head) * size + e;
  const size_t stride = size_t(A.heads) * size;
  constexpr int AHEAD = 8;      // parts requested together
  for (int p0 = 0; p0 < n; p0 += AHEAD) {
    float b[AHEAD];
#pragma unroll
    for (int i = 0; i < AHEAD; ++i) b[i] = p0 + i + 1 < n ? at[size_t(p0 + i) * stride] : 0.f;      // (the last piece left none)
#pragma unroll
    for (int i = 0; i < AHEAD; ++i) {
      if (p0 + i >= n) break;
      at[size_t(p0 + i) * stride] = cur;
      cur = fmaf(keep, cur, b[i]);
    }
  }
}

template <int DKP, int DVT, int CS, bool WIDE>
void launch_lightning(LightningArgs A, int S, hipStream_t s) {
  A.col_blocks = (A.dv + DVT - 1) / DVT;
  const dim3 grid(A.heads * A.col_blocks, S * A.pieces_per_seq);
  if (A.piece > 0) {
    lightning_kernel<DKP, DVT, CS, WIDE, true><<<grid, 256 * CS, 0, s>>>(A);
    lightning_pass_kernel<<<dim3((A.dk * A.dv + 255) / 256, A.heads, S), 256, 0, s>>>(A);
  }
  lightning_kernel<DKP, DVT, CS, WIDE, false><<<grid, 256 * CS, 0, s>>>(A);
}

}  // namespace kvcm

using namespace kvcm;

extern "C" {

// floats of scratch for a step of `rows` rows and S sequences walked in pieces
long long kvcm_lightning_carry_floats(int rows, int S, int heads, int dk, int dv, int piece) {
  if (piece <= 0 || rows < 0 || S < 0) return 0;
  return (static_cast<long long>(rows) / piece + S + 1) * heads * dk * dv;
}

// q, k [T, heads*dk], v [T, heads*dv] at their own strides; powers [heads, 66]: decay^0 .. decay^64 and decay^piece of every head;
// o [T, >= heads*dv]; state [slots, heads, dk, dv]; all 32-bit.  silu_in: q, k and v are silu of what is given.  piece (a
// multiple of 64): rows of a piece, with `carry` as scratch, where runs (max_run: the longest) are longer than that; 0: every run
// is one piece.
int kvcm_lightning(const float* q, int ldq, const float* k, int ldk, const float* v, int ldv, const float* powers, int silu_in, float* o,
                   int ldo, float* state, const int* run_start, const int* seq_start, const int* state_slots, int S, int heads, int dk,
                   int dv, int T, int piece, int max_run, float* carry, long long carry_floats, hipStream_t s) {
  if (S == 0 || T == 0) return 0;
  KVCM_REQUIRE(S > 0 && T > 0 && heads > 0 && dk > 0 && dv > 0 && max_run > 0, "lightning: bad sizes S=%d heads=%d dk=%d dv=%d", S, heads, dk, dv);
  KVCM_REQUIRE(dk <= 256, "lightning: a key size of %d is not supported (up to 256)", dk);
  KVCM_REQUIRE(ldq >= heads * dk && ldk >= heads * dk && ldv >= heads * dv && ldo >= heads * dv, "lightning: row strides too small");
  KVCM_REQUIRE(q && k && v && powers && o && state && run_start && seq_start && state_slots, "lightning: an operand is missing");
  KVCM_REQUIRE(piece >= 0 && piece % kLtRows == 0, "lightning: pieces of %d rows are not supported (a multiple of %d)", piece, kLtRows);
  LightningArgs A = {q, k, v, ldq, ldk, ldv, powers, o, ldo, state, run_start, seq_start, state_slots, heads, dk, dv, 1, silu_in, carry, 0, 1};
  if (piece > 0 && max_run > piece) {
    KVCM_REQUIRE(carry && carry_floats >= kvcm_lightning_carry_floats(T, S, heads, dk, dv, piece), "lightning: the scratch for the pieces is too small");
    A.piece = piece;
    A.pieces_per_seq = (max_run + piece - 1) / piece;
  }
  KVCM_REQUIRE(static_cast<long long>(S) * A.pieces_per_seq <= 65535 && heads <= 65535, "lightning: too many sequences and pieces for one launch");
  auto aligned = [](const void* x) { return reinterpret_cast<uintptr_t>(x) % 16 == 0; };
  const bool wide = dk % 4 == 0 && dv % 4 == 0 && ldq % 4 == 0 && ldk % 4 == 0 && ldv % 4 == 0 && aligned(q) && aligned(k) && aligned(v);
#define KVCM_LIGHTNING(DKP, DVT, CS)                          \
  {                                                           \
    if (wide) launch_lightning<DKP, DVT, CS, true>(A, S, s);  \
    else launch_lightning<DKP, DVT, CS, false>(A, S, s);      \
  }
  if (dk <= 64) { if (dv <= 32) KVCM_LIGHTNING(64, 32, 1) else KVCM_LIGHTNING(64, 64, 2) }
  else if (dk <= 128) { if (dv <= 32) KVCM_LIGHTNING(128, 32, 1) else if (dv <= 64) KVCM_LIGHTNING(128, 64, 2) else KVCM_LIGHTNING(128, 128, 2) }
  else KVCM_LIGHTNING(256, 32, 1)      // (wider stretches of values do not fit the local memory beside keys of this size)
#undef KVCM_LIGHTNING
  return launch_status("lightning");
}

}  // extern "C"
