// Two recurrences whose state is a matrix per head that decays by one number per head and token, S [dk, dv]:
//
//   delta 1 (the gated delta rule)    g = exp(-exp(a_log) softplus(a + dt_bias)),  beta = sigmoid(b)
//       q <- q / sqrt(|q|^2 + 1e-6) * dk^(-1/2),  k <- k / sqrt(|k|^2 + 1e-6)
//       S <- g S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q
//   delta 0 (state-space duality)     dt = softplus(a + dt_bias)
//       S <- exp(-exp(a_log) dt) S + dt k v^T;  o = S^T q + d_skip v
//
// q and k come in `groups` heads of dk entries, v in `heads` heads of dv; head h reads group h / (heads / groups).  Everything
// here is 32-bit.  A run that starts at position 0 starts from zero without reading its slot.
//
// The walk takes one token after another.  A value column j of S needs S^T k of its own column only, so columns are spread
// over lanes and workgroups (256 / G of them a workgroup, the key dimension of a column over G lanes); the tokens' vectors
// are staged through LDS a few at a time, the next ones requested before the current are computed, and a token's scalars
// (decay, rate, the lengths of its q and k) are made as its vectors are staged, so that no transcendental function and no
// sum across the head sits in the chain from token to token.
//
// Long runs are walked in pieces of L rows, all pieces at once.  A piece maps the state that enters it to the state that
// leaves it by S -> A S + B (both recurrences are linear in S): B is the piece walked from zero, A is the product of its
// decays, or, for the delta rule, the dk x dk matrix that the same walk makes of the identity when its values are zero: dk
// further columns beside the dv.  Three launches: every piece's A and B; the states that enter the pieces, one after another
// (a small product each); every piece again from the state that enters it, now with outputs.
#include "common.h"
#include "kvcm_hip.h"

namespace kvcm {

__device__ __forceinline__ float softplus32(float z) { return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z))); }

struct StateArgs {
  const float *q, *k, *v, *a, *b;      // 32-bit rows
  int ldq, ldk, ldv, lda, ldb;
  const float *dt_bias, *a_log, *d_skip;
  float* o;
  int ldo;
  float* state;                        // [slots, heads, dk, dv]
  const int *run_start, *seq_start, *state_slots;
  int heads, groups, dk, dv, col_blocks;
  float* carry;                        // pieces: per (piece, head) [dk][W] with W = dv + dk (delta) or dv, then per (piece, head) the decay
  int piece, pieces_per_seq, total_pieces;
};

// which rows of sequence s piece number p covers, and where its carry lies (pieces of all sequences are numbered so that no
// two meet: a sequence starts at floor(its first row / piece) + its own number)
__device__ __forceinline__ int piece_place(int run0, int s, int p, int piece) { return run0 / piece + s + p; }

// ENDS: the first of the three launches (no outputs, a state of W columns from zero / identity, written to the carry)
template <int DKP, int G, int TILE, bool DELTA, bool ENDS>
__global__ void __launch_bounds__(256) gated_state_kernel(StateArgs A) {
  constexpr int IPT = DKP / G, CB = 256 / G, V = 2 * DKP + CB, SC = 4;
  constexpr int PF = (TILE * V + 255) / 256;
  __shared__ __attribute__((aligned(16))) float tile[TILE][V + SC];      // per token: q, k (zero beyond dk), v of these columns, scalars
  const int head = blockIdx.x / A.col_blocks, cb = blockIdx.x % A.col_blocks;
  const int s = blockIdx.y / A.pieces_per_seq, p = blockIdx.y % A.pieces_per_seq;
  const int dk = A.dk, dv = A.dv, W = ENDS && DELTA ? dv + dk : dv;
  const int g = threadIdx.x % G, jl = threadIdx.x / G, j = cb * CB + jl;
  int r0 = A.run_start[s], r1 = A.run_start[s + 1];
  const int slot = A.state_slots[s];
  const int run0 = r0, run1 = r1;
  const bool pieces = A.piece > 0;
  if (pieces) {
    r0 = run0 + p * A.piece;
    r1 = run1 - r0 < A.piece ? run1 : r0 + A.piece;
  }
  if (r1 <= r0) return;
  const bool last = r1 == run1;
  if (ENDS && (last || slot < 0)) return;      // nothing follows the last piece
  const bool owns = j < W;
  if (slot < 0) {
    if (owns && g == 0)
      for (int row = r0; row < r1; ++row) A.o[size_t(row) * A.ldo + size_t(head) * dv + j] = 0.f;
    return;
  }
  const int group = head / (A.heads / A.groups);
  const bool fresh = A.seq_start[s] == 0;
  float* st = A.state + ((size_t(slot) * A.heads + head) * dk) * dv + (owns ? j : 0);      // [i][j]
  const int CW = DELTA ? dv + dk : dv;                                                       // a carry's columns
  float* cst = nullptr;
  if (pieces) cst = A.carry + ((size_t(piece_place(run0, s, p, A.piece)) * A.heads + head) * dk) * CW + (owns ? j : 0);
  float S[IPT];
#pragma unroll
  for (int il = 0; il < IPT; ++il) {
    const int i = g * IPT + il;
    if constexpr (ENDS) S[il] = (DELTA && owns && i < dk && j - dv == i) ? 1.f : 0.f;
    else if (pieces) S[il] = (i < dk && owns) ? cst[size_t(i) * CW] : 0.f;
    else S[il] = (i < dk && owns && !fresh) ? st[size_t(i) * dv] : 0.f;
  }
  const float rate = -expf(A.a_log[head]), dtb = A.dt_bias[head];
  const float skip = DELTA ? 0.f : A.d_skip[head];
  const float q_scale = 1.0f / sqrtf(float(dk));
  float pf[PF], sa = 0.f, sb = 0.f;
  auto request = [&](int t0) {      // unconditional loads from clamped places, masked afterwards
#pragma unroll
    for (int n = 0; n < PF; ++n) {
      const int e = threadIdx.x + n * 256;
      const int t = e / V, off = e % V;
      const int row = t0 + t < r1 ? t0 + t : r1 - 1;
      const bool vec = off < 2 * DKP;
      const int i = off % DKP, jj = cb * CB + (off - 2 * DKP);
      const bool ok = t < TILE && t0 + t < r1 && (vec ? i < dk : jj < dv);
      const size_t col = size_t(group) * dk + (i < dk ? i : dk - 1);
      const size_t vcol = size_t(head) * dv + ((jj >= 0 && jj < dv) ? jj : 0);
      const float* src = !vec ? A.v + size_t(row) * A.ldv + vcol : off < DKP ? A.q + size_t(row) * A.ldq + col : A.k + size_t(row) * A.ldk + col;
      const float val = *src;
      pf[n] = ok ? val : 0.f;
    }
    const int t = threadIdx.x < TILE ? threadIdx.x : TILE - 1;
    const int row = t0 + t < r1 ? t0 + t : r1 - 1;
    sa = A.a[size_t(row) * A.lda + head];
    if constexpr (DELTA) sb = A.b[size_t(row) * A.ldb + head];
  };
  auto stage = [&]() {
#pragma unroll
    for (int n = 0; n < PF; ++n) {
      const int e = threadIdx.x + n * 256;
      if (e < TILE * V) tile[e / V][e % V] = pf[n];
    }
    if (threadIdx.x < TILE) {
      const float dt = softplus32(sa + dtb);
      tile[threadIdx.x][V] = expf(rate * dt);
      tile[threadIdx.x][V + 1] = DELTA ? 1.0f / (1.0f + expf(-sb)) : dt;
    }
    if constexpr (DELTA) {      // the lengths of the staged q and k: sixteen lanes a vector
      __syncthreads();
      const int vec = threadIdx.x / 16, l = threadIdx.x % 16;
      if (vec < 2 * TILE) {
        const float* x = &tile[vec / 2][(vec & 1) * DKP];
        float ss = 0.f;
#pragma unroll
        for (int i = 0; i < DKP / 16; ++i) ss = fmaf(x[l + i * 16], x[l + i * 16], ss);
        ss = group_sum<16>(ss);
        if (l == 0) tile[vec / 2][V + 2 + (vec & 1)] = (1.0f / sqrtf(ss + 1e-6f)) * ((vec & 1) ? 1.0f : q_scale);
      }
    }
  };
  float decay = 1.f;
  request(r0);
  stage();
  __syncthreads();
  for (int t0 = r0; t0 < r1; t0 += TILE) {
    const int nt = r1 - t0 < TILE ? r1 - t0 : TILE;
    const bool more = t0 + TILE < r1;
    if (more) request(t0 + TILE);
    for (int t = 0; t < nt; ++t) {
      const float* tv = tile[t];
      const float keep = tv[V], take = tv[V + 1], vj = tv[2 * DKP + jl];
      float kd[IPT];
#pragma unroll
      for (int il = 0; il < IPT; ++il) kd[il] = tv[DKP + g * IPT + il];
      float u;
      if constexpr (DELTA) {
        const float fk = tv[V + 3];
        float sk = 0.f;
#pragma unroll
        for (int il = 0; il < IPT; ++il) {
          S[il] *= keep;
          sk = fmaf(kd[il], S[il], sk);
        }
        sk = group_sum<G>(sk) * fk;
        u = take * (vj - sk) * fk;
      } else {
        u = take * vj;
#pragma unroll
        for (int il = 0; il < IPT; ++il) S[il] *= keep;
        if constexpr (ENDS) decay *= keep;
      }
      float acc = 0.f;
#pragma unroll
      for (int il = 0; il < IPT; ++il) {
        S[il] = fmaf(kd[il], u, S[il]);
        if constexpr (!ENDS) acc = fmaf(S[il], tv[g * IPT + il], acc);
      }
      if constexpr (!ENDS) {
        acc = group_sum<G>(acc);
        if (owns && g == 0) A.o[size_t(t0 + t) * A.ldo + size_t(head) * dv + j] = DELTA ? acc * tv[V + 2] : fmaf(skip, vj, acc);
      }
    }
    __syncthreads();
    if (more) stage();
    __syncthreads();
  }
  if constexpr (ENDS) {
#pragma unroll
    for (int il = 0; il < IPT; ++il) {
      const int i = g * IPT + il;
      if (i < dk && owns) cst[size_t(i) * CW] = S[il];
    }
    if (!DELTA && cb == 0 && threadIdx.x == 0)
      A.carry[size_t(A.total_pieces) * A.heads * dk * CW + size_t(piece_place(run0, s, p, A.piece)) * A.heads + head] = decay;
  } else if (last) {
#pragma unroll
    for (int il = 0; il < IPT; ++il) {
      const int i = g * IPT + il;
      if (i < dk && owns) st[size_t(i) * dv] = S[il];
    }
  }
}

// the states that enter a sequence's pieces, walked from its slot (or zero): carry[piece].B <- S, then S <- A S + B.
// grid (heads * column blocks of 16, sequences); S of these columns in LDS.
constexpr int kPassCols = 16;
template <bool DELTA>
__global__ void __launch_bounds__(256) gated_state_pass_kernel(StateArgs A) {
  extern __shared__ __attribute__((aligned(16))) float cur[];      // [2][dk][kPassCols]
  const int head = blockIdx.x / A.col_blocks, cb = blockIdx.x % A.col_blocks, s = blockIdx.y;
  const int dk = A.dk, dv = A.dv, CW = DELTA ? dv + dk : dv;
  const int run0 = A.run_start[s], len = A.run_start[s + 1] - run0, slot = A.state_slots[s];
  if (len <= 0 || slot < 0) return;
  const int n = (len + A.piece - 1) / A.piece;
  const int jl = threadIdx.x % kPassCols, j = cb * kPassCols + jl, jc = j < dv ? j : dv - 1;
  const bool fresh = A.seq_start[s] == 0;
  const float* st = A.state + (size_t(slot) * A.heads + head) * dk * dv;
  const float* decays = A.carry + size_t(A.total_pieces) * A.heads * dk * CW;
  float* now = cur;
  float* next = cur + dk * kPassCols;
  for (int i = threadIdx.x / kPassCols; i < dk; i += 256 / kPassCols) now[i * kPassCols + jl] = fresh ? 0.f : st[size_t(i) * dv + jc];
  __syncthreads();
  for (int p = 0; p < n; ++p) {
    const size_t place = size_t(piece_place(run0, s, p, A.piece)) * A.heads + head;
    float* c = A.carry + place * dk * CW;
    const float keep = !DELTA && p + 1 < n ? decays[place] : 0.f;
    for (int i = threadIdx.x / kPassCols; i < dk; i += 256 / kPassCols) {
      float* row = c + size_t(i) * CW;
      if (p + 1 < n) {
        float acc = row[jc];
        if constexpr (DELTA) {
          const float* a = row + dv;
#pragma unroll 8
          for (int m = 0; m < dk; ++m) acc = fmaf(a[m], now[m * kPassCols + jl], acc);
        } else {
          acc = fmaf(keep, now[i * kPassCols + jl], acc);
        }
        next[i * kPassCols + jl] = acc;
      }
      if (j < dv) row[j] = now[i * kPassCols + jl];      // (a thread reads and writes its own element of B; A is only read)
    }
    __syncthreads();
    float* t = now;
    now = next;
    next = t;
  }
}

template <int DKP, int G, int TILE, bool DELTA>
void launch_state(StateArgs A, int S, hipStream_t s) {
  constexpr int CB = 256 / G;
  if (A.piece == 0) {
    A.pieces_per_seq = 1;
    A.col_blocks = (A.dv + CB - 1) / CB;
    gated_state_kernel<DKP, G, TILE, DELTA, false><<<dim3(A.heads * A.col_blocks, S), 256, 0, s>>>(A);
    return;
  }
  const int W = DELTA ? A.dv + A.dk : A.dv;
  StateArgs E = A;
  E.col_blocks = (W + CB - 1) / CB;
  gated_state_kernel<DKP, G, TILE, DELTA, true><<<dim3(E.heads * E.col_blocks, S * A.pieces_per_seq), 256, 0, s>>>(E);
  E.col_blocks = (A.dv + kPassCols - 1) / kPassCols;
  gated_state_pass_kernel<DELTA><<<dim3(E.heads * E.col_blocks, S), 256, 2 * sizeof(float) * A.dk * kPassCols, s>>>(E);
  E.col_blocks = (A.dv + CB - 1) / CB;
  gated_state_kernel<DKP, G, TILE, DELTA, false><<<dim3(E.heads * E.col_blocks, S * A.pieces_per_seq), 256, 0, s>>>(E);
}

}  // namespace kvcm

using namespace kvcm;

extern "C" {

// floats of scratch for a step of `rows` rows and S sequences walked in pieces
long long kvcm_gated_state_carry_floats(int rows, int S, int heads, int dk, int dv, int delta, int piece) {
  if (piece <= 0 || rows < 0 || S < 0) return 0;
  const long long places = rows / piece + S + 1;
  return places * heads * (static_cast<long long>(dk) * (delta ? dv + dk : dv) + 1);
}

// q, k [T, groups*dk], v [T, heads*dv], a (and with delta b) [T, heads] at their own strides; dt_bias, a_log (and without delta
// d_skip) [heads]; o [T, >= heads*dv]; state [slots, heads, dk, dv]; all 32-bit.  piece > 0: runs (max_run: the longest) are
// walked in pieces of that many rows, with `carry` as scratch.
int kvcm_gated_state(const float* q, int ldq, const float* k, int ldk, const float* v, int ldv, const float* a, int lda, const float* b,
                     int ldb, const float* dt_bias, const float* a_log, const float* d_skip, int delta, float* o, int ldo, float* state,
                     const int* run_start, const int* seq_start, const int* state_slots, int S, int heads, int groups, int dk, int dv,
                     int T, int piece, int max_run, float* carry, long long carry_floats, hipStream_t s) {
  if (S == 0 || T == 0) return 0;
  KVCM_REQUIRE(S > 0 && T > 0 && heads > 0 && groups > 0 && dk > 0 && dv > 0, "gated_state: bad sizes S=%d heads=%d dk=%d dv=%d", S, heads, dk, dv);
  KVCM_REQUIRE(heads % groups == 0, "gated_state: %d heads are not a multiple of %d groups", heads, groups);
  KVCM_REQUIRE(dk <= 256, "gated_state: a key size of %d is not supported (up to 256)", dk);
  KVCM_REQUIRE(ldq >= groups * dk && ldk >= groups * dk && ldv >= heads * dv && lda >= heads && (!delta || ldb >= heads) && ldo >= heads * dv,
               "gated_state: row strides too small");
  KVCM_REQUIRE(q && k && v && a && dt_bias && a_log && o && state && (delta ? b != nullptr : d_skip != nullptr), "gated_state: an operand is missing");
  KVCM_REQUIRE(static_cast<long long>(heads) * ((dv + dk + 15) / 16) < (1ll << 31), "gated_state: too many heads");
  StateArgs A = {q, k, v, a, b, ldq, ldk, ldv, lda, ldb, dt_bias, a_log, d_skip, o, ldo, state, run_start, seq_start, state_slots,
                 heads, groups, dk, dv, 0, carry, piece, 1, 0};
  if (piece > 0) {
    KVCM_REQUIRE(max_run > 0 && carry && carry_floats >= kvcm_gated_state_carry_floats(T, S, heads, dk, dv, delta, piece),
                 "gated_state: the scratch for the pieces is too small");
    A.pieces_per_seq = (max_run + piece - 1) / piece;
    A.total_pieces = T / piece + S + 1;
  }
  KVCM_REQUIRE(static_cast<long long>(S) * A.pieces_per_seq <= 65535, "gated_state: too many sequences and pieces for one launch");
#define KVCM_STATE(DKP, G, TILE)                                    \
  {                                                                 \
    if (delta) launch_state<DKP, G, TILE, true>(A, S, s);           \
    else launch_state<DKP, G, TILE, false>(A, S, s);                \
  }
  if (dk <= 16) KVCM_STATE(16, 4, 8)
  else if (dk <= 32) KVCM_STATE(32, 8, 8)
  else if (dk <= 64) KVCM_STATE(64, 8, 8)
  else if (dk <= 128) KVCM_STATE(128, 16, 8)
  else KVCM_STATE(256, 16, 4)
#undef KVCM_STATE
  return launch_status("gated_state");
}

}  // extern "C"
